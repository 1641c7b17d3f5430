"""Every operator of the layer-stack pipeline alone, through the C ABI, against the plain float64 statement of its
mechanism, in fp32 and in bf16."""
import numpy as np
import pytest

torch = pytest.importorskip("torch")
pytestmark = pytest.mark.gpu

from nanoflow_amd import kernels as K  # noqa: E402
from oracle import stack_oracle as S  # noqa: E402

import stack_cases as cases  # noqa: E402

F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [F32, BF16]
TOL = {F32: 2e-5, BF16: 1.2e-2}          # of the result's root mean square


@pytest.fixture(scope="module", autouse=True)
def _gpu():
    assert torch.cuda.is_available()
    K.lib()


def dev(a, dtype=None):
    t = torch.from_numpy(np.ascontiguousarray(a)).cuda()
    return t if dtype is None else t.to(dtype)


def rounded(a, dtype):
    """The values a tensor of that type holds, as float64."""
    return torch.from_numpy(np.ascontiguousarray(a, dtype=np.float32)).to(dtype).double().numpy()


def host(t):
    torch.cuda.synchronize()
    return t.double().cpu().numpy()


def close(got, want, dtype, what="", factor=1.0):
    got = host(got) if torch.is_tensor(got) else got
    assert np.isfinite(got).all(), what
    err, scale = np.abs(got - want).max(), max(np.sqrt((want ** 2).mean()), 1e-9)
    peak = max(np.abs(want).max() / scale, 1.0)
    assert err <= TOL[dtype] * factor * scale * peak, f"{what}: off by {err:.3e}, rms {scale:.3e}, peak {peak:.1f}"


# ---------------------------------------------------------------- products

@pytest.mark.parametrize("M,N,Kd", [(1, 8, 8), (3, 40, 104), (64, 264, 1024), (130, 136, 2048), (300, 512, 1032), (700, 384, 264),
                                    (1100, 264, 8200)])
def test_products(M, N, Kd):
    rng = np.random.default_rng(M)
    a, b = rng.standard_normal((M, Kd)), rng.standard_normal((N, Kd)) / np.sqrt(Kd)
    ws = torch.empty(1 << 24, dtype=torch.float32, device="cuda")
    for dtype in DTYPES:
        want = rounded(a, dtype) @ rounded(b, dtype).T
        da, db = dev(a, dtype), dev(b, dtype)
        close(K.gemm_nk(da, db, workspace=ws), want, dtype, "plain")
        close(K.gemm_nk(da, db, squared_relu=True, workspace=ws), np.maximum(want, 0) ** 2, dtype, "squared relu")
        close(K.gemm_nk(da, db, act=K.ACT_SILU, workspace=ws), S.silu(want), dtype, "silu")
        bias = rng.standard_normal(N) * 2
        close(K.gemm_nk(da, db, bias=dev(bias, dtype), workspace=ws), want + rounded(bias, dtype), dtype, "bias")
        if dtype == BF16:
            for shares in (1, 16):
                p = K.gemm_nk_sums(da, db, shares)
                close(p.double().sum(0), want, F32, f"{p.shape[0]} shares", factor=4)


# ---------------------------------------------------------------- rows

@pytest.mark.parametrize("width,ld", [(104, 104), (52, 56), (1, 8), (2050, 2056), (9000, 9000)])
def test_row_operators(width, ld):
    rng = np.random.default_rng(width)
    T, eps = 37, 1e-3
    pad = lambda a: np.pad(a, [(0, 0)] * (a.ndim - 1) + [(0, ld - width)])
    w = rng.standard_normal(width)
    x = rng.standard_normal((T, width))
    for dtype in DTYPES:
        for shares in (1, 3):
            y = rng.standard_normal((shares, T, width))
            kinds = [(dev(pad(y), F32), y.astype(np.float32).astype(np.float64).sum(0))]
            if shares == 1:
                kinds.append((dev(pad(y[0]), BF16), rounded(y[0], BF16)))
            for dy, vy in kinds:
                dx, act = dev(pad(x), F32), torch.full((T, ld), 7.0, dtype=dtype, device="cuda")
                K.norm_add_rows(dy, dev(pad(w), F32), dx, act, width, eps)
                want = x + S.rms_norm(vy, eps, w)
                close(dx[:, :width], want, F32)
                close(act[:, :width], want, dtype)
                assert not host(act[:, width:]).any() and not host(dx[:, width:]).any()
        index = np.array([5, 0, 36, 5], np.int32)
        got = K.gather_norm_rows(dev(pad(x), F32), dev(index), dev(pad(w), F32), width, eps, dtype)
        close(got[:, :width], S.rms_norm(x[index], eps, w), dtype)
        table, pos = rng.standard_normal((9, width)), rng.standard_normal((50, width))
        tok, at = rng.integers(0, 9, T).astype(np.int32), rng.integers(0, 50, T).astype(np.int32)
        gx, ga = K.embed_rows(dev(tok), dev(at), dev(pad(table), dtype), dev(pad(pos), dtype))
        want = rounded(table, dtype)[tok] + rounded(pos, dtype)[at]
        close(gx[:, :width], want, F32)
        close(ga[:, :width], want, dtype)
        gx, _ = K.embed_rows(dev(tok), dev(at), dev(pad(table), dtype), None)
        close(gx[:, :width], rounded(table, dtype)[tok], F32)


def test_token_shift_reads_the_row_before_the_state_or_nothing():
    rng = np.random.default_rng(0)
    b = cases.batch([9, 0, 30], [(0, 5), (7, 3), (16, 1)], seed=3)
    width, slots = 40, np.array([4, 0, 2, 5, 1, 3], np.int32)
    x, state, mu = rng.standard_normal((b.tokens, width)), rng.standard_normal((6, width)), rng.random((5, width))
    prev = np.empty_like(x)
    for r in range(b.req_num):
        i0, i1 = b.input_indptr[r:r + 2]
        first = 0 if b.per_token_offset[i0] == 0 else state[slots[r]]
        prev[i0:i1] = np.vstack([np.broadcast_to(first, (1, width)), x[i0:i1 - 1]])
    for dtype in DTYPES:
        got = K.token_shift(dev(x, F32), dev(state, F32), dev(mu, F32), dev(b.input_indptr), dev(b.rev_input_indptr),
                            dev(b.per_token_offset), dev(slots), dtype)
        close(got, x + (prev - x) * mu[:, None], dtype)


def test_tanh_and_argmax():
    rng = np.random.default_rng(0)
    p = rng.standard_normal((4, 19, 24)) * 2
    for dtype in DTYPES:
        close(K.tanh_rows(dev(p, F32), dtype), np.tanh(p.sum(0)), dtype)
    l = rng.standard_normal((7, 1500)).astype(np.float32)
    l[2, [3, 700, 1499]] = 9.0                       # the smallest column wins
    l[4] = -np.inf
    l[5, 1499] = 11.0                                # beyond the true width
    got = host(K.argmax_f32(dev(l), cols=1499)).astype(int)
    want = l[:, :1499].argmax(1)
    assert got.tolist() == want.tolist() and got[2] == 3


# ---------------------------------------------------------------- attention

def table_of(positions, dims, base):
    i = np.arange(dims // 2)
    a = np.arange(positions)[:, None] * base ** (-2.0 * i / dims)
    return dev(np.stack([np.cos(a), np.sin(a)], -1), F32)


def device_batch(b):
    return {"input_indptr": dev(b.input_indptr), "kv_indptr": dev(b.kv_indptr), "kv_indices": dev(b.kv_indices),
            "rev_input_indptr": dev(b.rev_input_indptr), "positions": dev(b.per_token_offset)}


def append(layout, b, proj, pool, q_norm=None, k_norm=None, rot=None, eps=1e-5):
    d = device_batch(b)
    H, G, dim, vdim = layout.heads, layout.kv_heads, layout.dim, layout.vdim
    return K.qkv_append(layout, proj, (0, H * dim, (H + G) * dim), q_norm, k_norm, eps, rot or K.rotation(), pool,
                        d["kv_indptr"], d["kv_indices"], d["rev_input_indptr"], d["positions"])


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,rot_dims,interleaved", [
    (4, 2, 64, 64, 64, True), (4, 2, 64, 64, 32, False), (3, 1, 18, 10, 6, True), (2, 2, 20, 36, 20, False), (1, 1, 256, 256, 128, True),
    (6, 3, 96, 32, 0, True), (5, 5, 12, 16, 10, True)])
def test_norm_rotation_and_append(heads, kv_heads, dim, vdim, rot_dims, interleaved):
    rng = np.random.default_rng(dim)
    b = cases.batch([40, 3], [(0, 37), (21, 30), (5, 2)], seed=dim)
    cols = heads * dim + kv_heads * (dim + vdim)
    proj = rng.standard_normal((b.tokens, cols + 4))
    qn, kn = rng.standard_normal(dim), rng.standard_normal(dim)
    tab = table_of(80, rot_dims, 50.0) if rot_dims else None
    for dtype in DTYPES:
        layout = K.kv_layout(dtype, heads, kv_heads, dim, vdim)
        pool = K.kv_pool(layout, b.num_pages)
        q = append(layout, b, dev(proj, dtype), pool, dev(qn, F32), dev(kn, F32), K.rotation(tab, rot_dims, interleaved))
        v = rounded(proj, dtype)
        pos = b.per_token_offset
        heads_of = lambda at, n, d: v[:, at:at + n * d].reshape(-1, n, d)
        want_q = S.rotate(S.rms_norm(heads_of(0, heads, dim), 1e-5, qn), pos, rot_dims, 50.0, interleaved)
        want_k = S.rotate(S.rms_norm(heads_of(heads * dim, kv_heads, dim), 1e-5, kn), pos, rot_dims, 50.0, interleaved)
        want_v = heads_of((heads + kv_heads) * dim, kv_heads, vdim)
        close(q[:, :, :dim], want_q, dtype)
        assert not host(q[:, :, dim:]).any()
        kp, vp = layout.k_pad, layout.v_pad
        pages = host(pool)
        pk = pages[:, :kv_heads * 16 * kp].reshape(-1, kv_heads, 16, kp)
        pv = pages[:, kv_heads * 16 * kp:].reshape(-1, kv_heads, vp, 16)
        page = b.kv_indices[b.kv_indptr[b.rev_input_indptr] + pos // 16]
        close(pk[page, :, pos % 16][:, :, :dim], want_k, dtype)
        assert np.array_equal(pv[page, :, :, pos % 16][:, :, :vdim], want_v)        # values are copied
        touched = np.zeros((b.num_pages, 16), bool)
        touched[page, pos % 16] = True
        assert not pk.transpose(0, 2, 1, 3)[~touched].any() and not pv.transpose(0, 3, 1, 2)[~touched].any()


def attention_case(dtype, heads, kv_heads, dim, vdim, window, keep, b, n_decode, seed=0, mark=None, scale=None, out_scale=1.0, gate=None, softcap=None):
    """Histories and the batch through append and attention; the plain result for the batch's rows.
    mark: list of (request, query position, key position): that key is made to stand out for that query."""
    rng = np.random.default_rng(seed)
    scale = dim ** -0.5 if scale is None else scale
    cols = heads * dim + kv_heads * (dim + vdim)
    full = [rng.standard_normal((int(n), cols)) for n in b.kv_len]
    for r, p, j in mark or []:
        key = full[r][j, heads * dim:(heads + kv_heads) * dim].reshape(kv_heads, dim)
        key *= 3.0
        full[r][p, :heads * dim] = np.repeat(key, heads // kv_heads, 0).ravel() * (14.0 / (9.0 * dim * scale))
    sink = rng.standard_normal(heads)
    layout = K.kv_layout(dtype, heads, kv_heads, dim, vdim)
    pool = K.kv_pool(layout, b.num_pages)
    h, reqs = cases.history_batch(b)
    if h is not None:
        append(layout, h, dev(np.concatenate([full[r][:len_] for r, len_ in zip(reqs, np.diff(h.input_indptr))]), dtype), pool)
    rows = np.concatenate([full[r][b.kv_len[r] - n:] for r, n in enumerate(np.diff(b.input_indptr))])
    q = append(layout, b, dev(rows, dtype), pool)
    got = K.window_attention(layout, q, pool, device_batch(b), window=window, keep_first=keep, scale=scale, sink=dev(sink, F32),
                             out_scale=out_scale, decode=n_decode, gate=None if gate is None else dev(gate, dtype), softcap=softcap or 0.0)
    want = []
    for r, n in enumerate(np.diff(b.input_indptr)):
        v = rounded(full[r], dtype)
        T = len(v)
        cut = lambda at, m, d: v[:, at:at + m * d].reshape(T, m, d)
        mask = S.window_mask(T, window or 10 ** 9, keep)
        o = S.sink_attention(cut(0, heads, dim), cut(heads * dim, kv_heads, dim), cut((heads + kv_heads) * dim, kv_heads, vdim), mask,
                             scale, sink.astype(np.float32), softcap)
        want.append(o[T - n:].reshape(n, -1))
    return got, np.concatenate(want) * out_scale


@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(4, 2, 64, 64), (6, 2, 32, 48), (5, 1, 18, 10), (20, 1, 16, 16), (3, 3, 128, 96),
                                                     (2, 1, 160, 256), (40, 2, 8, 24)])
@pytest.mark.parametrize("window,keep", [(24, 5), (1, 0), (64, 33), (0, 0), (200, 16), (7, 40)])
def test_window_attention(heads, kv_heads, dim, vdim, window, keep):
    b = cases.batch([0, 95, 128, 31], [(0, 70), (50, 41), (33, 2), (0, 1), (112, 16)], seed=window)
    for dtype in DTYPES:
        got, want = attention_case(dtype, heads, kv_heads, dim, vdim, window, keep, b, 4, seed=dim, out_scale=1.3)
        close(got, want, dtype, f"{dtype}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("query", [47, 48, 63, 64, 90, 127])
def test_a_key_at_the_windows_edge(dtype, query):
    """One key scores far above the others: just inside and just outside the window, among the kept first positions and just
    after them, at page borders; in a prompt and decoded."""
    window, keep = 32, 6
    for key in sorted({query - window + 1, query - window, keep - 1, keep, 15, 16, 31, 32, query - 1, query}):
        if not 0 <= key <= query:
            continue
        for b, n_decode in ((cases.batch([query], [], seed=key), 1), (cases.batch([], [(0, query + 1)], seed=key), 0),
                            (cases.batch([], [(query - 1, 2)], seed=key), 0)):
            got, want = attention_case(dtype, 4, 2, 32, 32, window, keep, b, n_decode, seed=key, mark=[(0, query, key)])
            close(got[-1], want[-1], dtype, f"key {key} decode {n_decode}")


@pytest.mark.parametrize("scale", [0.0, -0.3])
def test_scales_that_are_not_positive(scale):
    b = cases.batch([40], [(0, 50)], seed=2)
    for dtype in DTYPES:
        got, want = attention_case(dtype, 4, 2, 32, 32, 20, 3, b, 1, seed=1, scale=scale)
        close(got, want, dtype)


def test_long_decode_context_and_many_requests():
    b = cases.batch(np.random.default_rng(0).integers(1, 700, 80).tolist(), [], seed=1)
    got, want = attention_case(BF16, 8, 2, 64, 64, 300, 20, b, 80, seed=2)
    close(got, want, BF16)


# ---------------------------------------------------------------- recurrences

def recurrence_case(kind, dtype, heads, dim, vdim, b, n_decode, *, rot_dims=0, decay=None, z_shift=0.0, seed=0, slots=None, norm=True,
                    spike=None):
    """Histories and the batch through the operator; the plain result for the batch's rows and the states left behind."""
    rng = np.random.default_rng(seed)
    n_req, eps, k_scale, out_scale = b.req_num, 1e-4, dim ** -0.5, 0.8
    slots = np.random.default_rng(seed + 1).permutation(n_req + 2)[:n_req].astype(np.int32) if slots is None else slots
    qk, vg = heads * dim, heads * vdim
    full = [{"q": rng.standard_normal((n, qk)), "k": rng.standard_normal((n, qk)), "v": rng.standard_normal((n, vg)),
             "g": rng.standard_normal((n, vg)), "z": rng.standard_normal((n, qk)) + z_shift, "x": rng.standard_normal((n, 24))}
            for n in b.kv_len]
    if spike:                                                      # a key and a query that agree, far apart
        r, key, query = spike
        full[r]["k"][key] *= 6.0
        full[r]["q"][query] = full[r]["k"][key]
    w0, u, nw = rng.standard_normal(qk) - 3.0, rng.standard_normal((heads, dim)), rng.standard_normal(vg)
    decay = np.asarray(decay if decay is not None else np.linspace(0.3, 1.0, heads))
    state = torch.full((n_req + 2, heads * K.lib().nf_recurrence_state_elements(dim, vdim)), 5.0, dtype=F32, device="cuda")
    shift = torch.full((n_req + 2, 24), 5.0, dtype=F32, device="cuda")
    tab = table_of(int(b.kv_len.max()) + 1, rot_dims, 40.0) if rot_dims else None
    fixed = kind == K.FIXED_DECAY

    def run(batch, rows, sl, dec):
        cat = lambda key, dt: dev(np.concatenate([r[key] for r in rows]), dt)
        d = {"input_indptr": dev(batch.input_indptr), "positions": dev(batch.per_token_offset), "state_slots": dev(sl)}
        extra = dict(rot=K.rotation(tab, rot_dims), k_scale=k_scale, log2_decay=dev(np.log2(np.maximum(decay, 2.0 ** -126)), F32)) if fixed else \
            dict(z=cat("z", F32), w0=dev(w0, F32), u=dev(u, F32), shift_x=cat("x", F32), shift_state=shift)
        return K.linear_recurrence(kind, cat("q", dtype), cat("k", dtype), cat("v", dtype), cat("g", dtype), heads, dim, vdim, state, d,
                                   eps=eps, decode=dec, norm_weight=dev(nw, F32) if norm else None, out_scale=out_scale, **extra)

    h, reqs = cases.history_batch(b)
    if h is not None:
        run(h, [{k: v[:n] for k, v in full[r].items()} for r, n in zip(reqs, np.diff(h.input_indptr))], slots[reqs], 0)
    got = run(b, [{k: v[b.kv_len[r] - n:] for k, v in full[r].items()} for r, n in enumerate(np.diff(b.input_indptr))], slots, n_decode)
    want = []
    for r, n in enumerate(np.diff(b.input_indptr)):
        T = int(b.kv_len[r])
        q, k, v, g = (rounded(full[r][s], dtype) for s in "qkvg")
        q, k, v = q.reshape(T, heads, dim), k.reshape(T, heads, dim), v.reshape(T, heads, vdim)
        if fixed:
            pos = np.arange(T)
            o = S.fixed_decay_recurrence(S.rotate(q, pos, rot_dims, 40.0, False), S.rotate(k, pos, rot_dims, 40.0, False) * k_scale, v, decay)
        else:
            w = np.exp(-np.exp(full[r]["z"] + w0)).reshape(T, heads, dim)
            o = S.bonus_recurrence(q, k, v, w, u)
        y = S.rms_norm(o, eps).reshape(T, -1) * S.silu(g) * (nw if norm else 1.0) * out_scale
        want.append(y[T - n:])
        if not fixed:
            np.testing.assert_array_equal(host(shift[int(slots[r])]).astype(np.float32), full[r]["x"][-1].astype(np.float32))
    unused = [s for s in range(n_req + 2) if s not in slots.tolist()]
    assert (host(state[unused]) == 5.0).all()
    return got, np.concatenate(want)


SHAPES = [(2, 64, 64), (3, 32, 48), (2, 20, 36), (1, 128, 128), (2, 10, 6), (1, 16, 16), (3, 48, 80), (1, 160, 256)]


@pytest.mark.parametrize("heads,dim,vdim", SHAPES)
@pytest.mark.parametrize("kind", [K.FIXED_DECAY, K.TOKEN_DECAY])
def test_recurrences(kind, heads, dim, vdim):
    """Decode rows and portions of every length beside each other: in chunks (long portions), row by row (short ones)."""
    for decode, portions in (([7, 0, 100], [(0, 150), (33, 64), (16, 17), (0, 65)]), ([5], [(0, 2), (40, 3), (9, 1)]), ([], [(10, 300)])):
        b = cases.batch(decode, portions, seed=dim)
        for dtype in DTYPES:
            got, want = recurrence_case(kind, dtype, heads, dim, vdim, b, len(decode), seed=dim, rot_dims=(dim // 2) // 2 * 2, norm=dim != 64)
            close(got, want, dtype, f"{dtype} {decode} {portions}", factor=4 if dtype == F32 else 1)


@pytest.mark.parametrize("z_shift", [-6.0, 1.5, 4.0, 7.0])
def test_token_decays_from_almost_one_to_nothing(z_shift):
    b = cases.batch([20], [(0, 130), (17, 40)], seed=5)
    for dtype in DTYPES:
        got, want = recurrence_case(K.TOKEN_DECAY, dtype, 2, 64, 64, b, 1, z_shift=z_shift, seed=3)
        close(got, want, dtype, factor=8 if dtype == F32 else 1)


@pytest.mark.parametrize("decay", [[1.0, 0.999], [1e-6, 0.02], [0.5, 0.0]])
def test_fixed_decays_from_one_to_nothing(decay):
    b = cases.batch([20], [(0, 130), (17, 40)], seed=6)
    for dtype in DTYPES:
        got, want = recurrence_case(K.FIXED_DECAY, dtype, 2, 32, 32, b, 1, decay=decay, rot_dims=32, seed=4)
        close(got, want, dtype, factor=4 if dtype == F32 else 1)


@pytest.mark.parametrize("kind", [K.FIXED_DECAY, K.TOKEN_DECAY])
@pytest.mark.parametrize("key,query", [(0, 63), (0, 64), (63, 64), (15, 16), (16, 31), (127, 128), (3, 199), (199, 199), (0, 0)])
def test_a_key_far_back_is_found(kind, key, query):
    """A key that answers one query among many, across the borders of steps and chunks, in a prompt, cut before the query, and
    decoded."""
    for b, n_decode in ((cases.batch([], [(0, 200)], seed=1), 0), (cases.batch([query], [], seed=2), 1),
                        (cases.batch([], [(max(query - 1, 0), 40)], seed=3), 0)):
        if query >= b.kv_len[0]:
            continue
        got, want = recurrence_case(kind, BF16, 1, 64, 64, b, n_decode, decay=[0.999], z_shift=-4.0, seed=7, spike=(0, key, query))
        close(got, want, BF16, f"decode {n_decode}")


@pytest.mark.parametrize("heads,dim,vdim", [(2, 64, 64), (3, 20, 36), (1, 160, 256)])
def test_fixed_decay_without_norm_and_gate(heads, dim, vdim):
    """What the recurrence leaves when its heads are normed together later: the plain sums, scaled."""
    rng = np.random.default_rng(dim)
    b = cases.batch([7, 0], [(0, 150), (16, 3)], seed=1)
    decay = np.linspace(0.4, 1.0, heads)
    for dtype in DTYPES:
        state = torch.full((b.req_num, heads * K.lib().nf_recurrence_state_elements(dim, vdim)), 5.0, dtype=F32, device="cuda")
        full = [{"q": rng.standard_normal((n, heads * dim)), "k": rng.standard_normal((n, heads * dim)) / dim, "v": rng.standard_normal((n, heads * vdim))}
                for n in b.kv_len]
        slots = np.arange(b.req_num, dtype=np.int32)[::-1].copy()

        def run(batch, rows, sl, dec):
            cat = lambda key: dev(np.concatenate([r[key] for r in rows]), dtype)
            d = {"input_indptr": dev(batch.input_indptr), "positions": dev(batch.per_token_offset), "state_slots": dev(sl)}
            return K.linear_recurrence(K.FIXED_DECAY, cat("q"), cat("k"), cat("v"), None, heads, dim, vdim, state, d, eps=1.0, decode=dec,
                                       log2_decay=dev(np.log2(decay), F32), out_scale=0.5)

        h, reqs = cases.history_batch(b)
        run(h, [{k: v[:n] for k, v in full[r].items()} for r, n in zip(reqs, np.diff(h.input_indptr))], slots[reqs], 0)
        got = run(b, [{k: v[b.kv_len[r] - n:] for k, v in full[r].items()} for r, n in enumerate(np.diff(b.input_indptr))], slots, 2)
        want = []
        for r, n in enumerate(np.diff(b.input_indptr)):
            T = int(b.kv_len[r])
            q, k, v = (rounded(full[r][s], dtype).reshape(T, heads, -1) for s in "qkv")
            want.append(S.fixed_decay_recurrence(q, k, v, decay)[T - n:].reshape(n, -1) * 0.5)
        close(got, np.concatenate(want), dtype, str(dtype), factor=4 if dtype == F32 else 1)
