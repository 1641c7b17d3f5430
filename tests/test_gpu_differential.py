"""Operators of layer-stack models with two attention maps per head, short convolutions, capped scores, windows over latents and
experts in groups, each alone through the C ABI against the plain float64 statement of its mechanism, in fp32 and in bf16."""
import numpy as np
import pytest

torch = pytest.importorskip("torch")
pytestmark = pytest.mark.gpu

from nanoflow_amd import kernels as K, synth  # noqa: E402
from oracle import stack_oracle as S  # noqa: E402

import stack_cases as cases  # noqa: E402
from test_gpu_latent_and_mixture import check_routing, latent_case, padded  # noqa: E402
from test_gpu_stack_kernels import BF16, DTYPES, F32, attention_case, close, dev, device_batch, host, rounded, table_of  # noqa: E402


@pytest.fixture(scope="module", autouse=True)
def _gpu():
    assert torch.cuda.is_available()
    K.lib()


# ---------------------------------------------------------------- short convolution, rotation, append

@pytest.mark.parametrize("heads,kv_heads,dim,vdim,maps,rot,taps", [(4, 2, 64, 128, 2, 64, 3), (6, 2, 24, 40, 2, 16, 4), (3, 1, 18, 10, 2, 6, 2),
                                                                   (2, 2, 20, 36, 1, 0, 5), (1, 1, 8, 8, 2, 8, 1), (5, 5, 7, 9, 1, 4, 9),
                                                                   (2, 1, 160, 256, 2, 32, 3)])
def test_convolution_rotation_and_append_in_portions(heads, kv_heads, dim, vdim, maps, rot, taps):
    """Sequences of several requests in portions of every size from one token on; the slots held something else before."""
    rng = np.random.default_rng(dim)
    qn, kn = heads * maps * dim, kv_heads * maps * dim
    cols = qn + kn + kv_heads * vdim
    ld, lengths, slots = (cols + 7) // 8 * 8, [41, 30, 12], np.array([2, 0, 3], np.int32)
    full = [rng.standard_normal((n, ld)) for n in lengths]
    w = rng.standard_normal((cols, taps))
    table = table_of(60, rot, 50.0) if rot else None
    portions = [[7, 1, 1], [1, 2, 1], [2, 1, 3], [3, 17, 1], [1, 1, 1], [16, 1, 2], [1, 5, 1], [10, 2, 2]]
    assert np.array(portions).sum(0).tolist() == lengths
    for dtype in DTYPES:
        layout = K.kv_layout(dtype, heads, kv_heads, dim, vdim, maps)
        state = torch.full((5, max(taps - 1, 1), ld), 77.0, dtype=dtype, device="cuda")
        weight = dev(padded(w.T, ld), dtype)
        pages = [np.arange(4 * r, 4 * r + 4) for r in range(3)]
        pool = K.kv_pool(layout, 12)
        at, queries = [0, 0, 0], [[], [], []]
        for counts in portions:
            b = synth.make_batch([], [(at[r], counts[r]) for r in range(3)], vocab=10, seed=0)
            used = np.diff(b.kv_indptr)
            b.kv_indices = np.concatenate([pages[r][:used[r]] for r in range(3)]).astype(np.int32)
            d = device_batch(b)
            proj = dev(np.concatenate([full[r][at[r]:at[r] + counts[r]] for r in range(3)]), dtype)
            conv = K.short_conv(weight, state, d["input_indptr"], dev(slots))
            q = host(K.qkv_append(layout, proj, (0, qn, qn + kn), None, None, 1e-5, K.rotation(table, rot), pool, d["kv_indptr"], d["kv_indices"],
                                  d["rev_input_indptr"], d["positions"], conv=conv))
            assert not q[:, :, dim:].any()
            for r in range(3):
                first = b.input_indptr[r]
                queries[r].append(q[first:first + counts[r], :, :dim])
                at[r] += counts[r]
        held = host(pool)
        split = kv_heads * maps * 16 * layout.k_pad
        pk = held[:, :split].reshape(-1, kv_heads * maps, 16, layout.k_pad)
        pv = held[:, split:].reshape(-1, kv_heads, layout.v_pad, 16)
        for r, n in enumerate(lengths):
            y = S.short_conv(rounded(full[r], dtype)[:, :cols], rounded(w, dtype))
            pos = np.arange(n)
            turn = lambda x: S.rotate(x.reshape(n, -1, dim), pos, rot, 50.0, False)
            close(np.concatenate(queries[r]), turn(y[:, :qn]), dtype, f"queries {r}")
            page = pages[r][pos // 16]
            close(pk[page, :, pos % 16][:, :, :dim], turn(y[:, qn:qn + kn]), dtype, f"keys {r}")
            close(pv[page, :, :, pos % 16][:, :, :vdim], y[:, qn + kn:].reshape(n, kv_heads, vdim), dtype, f"values {r}")
        for slot in (1, 4):
            assert (host(state)[slot] == 77.0).all()                         # no one else's slot is touched


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,maps,rot,taps", [(4, 2, 64, 128, 2, 64, 4), (3, 1, 24, 40, 2, 16, 3), (2, 1, 100, 72, 1, 48, 6),
                                                                   (1, 1, 160, 256, 2, 32, 2), (2, 2, 16, 16, 1, 8, 0)])
def test_many_rows_are_the_rows_of_small_portions(heads, kv_heads, dim, vdim, maps, rot, taps):
    """More than a thousand rows of unequal requests at a time, single tokens between them, against the same a few tokens at a time: the
    same bits, whatever rows a workgroup has beside each other."""
    rng = np.random.default_rng(taps)
    qn, kn = heads * maps * dim, kv_heads * maps * dim
    ld, lengths = (qn + kn + kv_heads * vdim + 7) // 8 * 8, [701, 2, 333, 1, 47, 515, 5]
    n, cuts = len(lengths), [[120, 1, 333, 0, 46, 515, 2], [581, 1, 0, 1, 1, 0, 3]]      # 1017 rows in the first, few in the second
    cuts = [[a + (9 if r == 0 else 0) for r, a in enumerate(cuts[0])], [a - (9 if r == 0 else 0) for r, a in enumerate(cuts[1])]]
    assert sum(cuts[0]) >= 1024 and (np.array(cuts).sum(0) == lengths).all()
    full = [rng.standard_normal((t, ld)) for t in lengths]
    w, table = rng.standard_normal((max(taps, 1), ld)), table_of(800, rot, 50.0)
    pages = np.split(rng.permutation(sum(-(-t // 16) for t in lengths)), np.cumsum([-(-t // 16) for t in lengths])[:-1])

    def run(dtype, steps):
        layout = K.kv_layout(dtype, heads, kv_heads, dim, vdim, maps)
        state = torch.full((n, max(taps - 1, 1), ld), 77.0, dtype=dtype, device="cuda")
        pool, at, queries = K.kv_pool(layout, sum(map(len, pages))), [0] * n, [[] for _ in range(n)]
        for counts in steps:
            live = [r for r in range(n) if counts[r]]
            b = synth.make_batch([], [(at[r], counts[r]) for r in live], vocab=10, seed=0)
            b.kv_indices = np.concatenate([pages[r][:used] for r, used in zip(live, np.diff(b.kv_indptr))]).astype(np.int32)
            d, slots = device_batch(b), dev(np.array(live, np.int32))
            conv = K.short_conv(dev(w, dtype), state, d["input_indptr"], slots) if taps else None
            proj = dev(np.concatenate([full[r][at[r]:at[r] + counts[r]] for r in live]), dtype)
            q = host(K.qkv_append(layout, proj, (0, qn, qn + kn), None, None, 1e-5, K.rotation(table, rot), pool, d["kv_indptr"], d["kv_indices"],
                                  d["rev_input_indptr"], d["positions"], conv=conv))
            for i, r in enumerate(live):
                queries[r].append(q[b.input_indptr[i]:b.input_indptr[i + 1]])
                at[r] += counts[r]
        return [np.concatenate(q) for q in queries], host(pool)

    pieces = []
    left = list(lengths)
    while any(left):
        pieces.append([min(t, 3 + (7 * r + 5 * len(pieces)) % 90) for r, t in enumerate(left)])
        left = [a - c for a, c in zip(left, pieces[-1])]
    assert max(map(sum, pieces)) < 1024
    for dtype in DTYPES:
        many, few = run(dtype, cuts), run(dtype, pieces)
        for a, b in zip(many[0], few[0]):
            assert np.array_equal(a, b)
        assert np.array_equal(many[1], few[1])
        r = 0
        y = rounded(full[r], dtype)[:, :qn]
        if taps:
            y = S.short_conv(y, rounded(w.T[:qn], dtype))
        close(many[0][r][:, :, :dim], S.rotate(y.reshape(lengths[r], -1, dim), np.arange(lengths[r]), rot, 50.0, False), dtype)


# ---------------------------------------------------------------- two maps, capped scores

def maps_case(dtype, heads, kv_heads, dim, vdim, window, b, n_decode, seed=0, mark=None, scale=None, cap=5.0, weight=0.45, eps=1e-5, diff=0.3):
    """Histories and the batch through append and attention; the plain result for the batch's rows.  mark: (request, query position,
    key position, map): that map's key is made to stand out for that query."""
    rng = np.random.default_rng(seed)
    scale = dim ** -0.5 if scale is None else scale
    qn, kn = heads * 2 * dim, kv_heads * 2 * dim
    cols = qn + kn + kv_heads * vdim
    full = [rng.standard_normal((int(n), (cols + 7) // 8 * 8)) for n in b.kv_len]
    if mark:
        r, p, j, m = mark
        keys = full[r][j, qn:qn + kn].reshape(kv_heads, 2, dim)
        keys[:, m] *= 3.0 * np.sqrt(dim) / np.linalg.norm(keys[:, m], axis=-1, keepdims=True)
        full[r][p, :qn].reshape(heads, 2, dim)[:, m] = np.repeat(keys[:, m], heads // kv_heads, 0) * (14.0 / (9.0 * dim * scale))
    layout = K.kv_layout(dtype, heads, kv_heads, dim, vdim, 2)
    pool = K.kv_pool(layout, b.num_pages)

    def append(batch, rows):
        d = device_batch(batch)
        return K.qkv_append(layout, dev(np.concatenate(rows), dtype), (0, qn, qn + kn), None, None, eps, K.rotation(), pool, d["kv_indptr"],
                            d["kv_indices"], d["rev_input_indptr"], d["positions"])

    h, reqs = cases.history_batch(b)
    if h is not None:
        append(h, [full[r][:n] for r, n in zip(reqs, np.diff(h.input_indptr))])
    lens = np.diff(b.input_indptr)
    q = append(b, [full[r][len(full[r]) - n:] for r, n in enumerate(lens)])
    got = K.window_attention(layout, q, pool, device_batch(b), window=window, keep_first=0, scale=scale, decode=n_decode, out_scale=1.0 - diff,
                             softcap=cap or 0.0, map_weight=weight, head_eps=eps)
    want = []
    for r, n in enumerate(lens):
        v = rounded(full[r], dtype)
        T = len(v)
        o = S.differential_attention(v[:, :qn].reshape(T, heads, 2, dim), v[:, qn:qn + kn].reshape(T, kv_heads, 2, dim),
                                     v[:, qn + kn:cols].reshape(T, kv_heads, vdim), S.window_mask(T, window or T + 1, 0), scale, cap, weight, diff, eps)
        want.append(o[T - n:].reshape(n, -1))
    return got, np.concatenate(want)


@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(4, 2, 64, 128), (6, 2, 32, 48), (5, 1, 18, 10), (20, 1, 16, 64), (3, 3, 128, 96), (2, 1, 160, 256),
                                                     (4, 4, 64, 64), (2, 2, 128, 128), (8, 2, 100, 256), (40, 2, 8, 24)])
@pytest.mark.parametrize("window", [24, 1, 64, 0, 200])
def test_difference_of_two_maps(heads, kv_heads, dim, vdim, window):
    b = cases.batch([0, 95, 128, 31], [(0, 70), (50, 41), (33, 2), (0, 1), (112, 16)], seed=window)
    for dtype in DTYPES:
        # a row that sees one key only is (1 - weight) v before its norm, whatever the scores are
        got, want = maps_case(dtype, heads, kv_heads, dim, vdim, window, b, 4, seed=dim)
        close(got, want, dtype, f"{dtype}", factor=1.5)


@pytest.mark.parametrize("cap,scale,weight,diff", [(None, 0.3, 0.2, 0.8), (0.5, 0.3, 1.4, 0.0), (50.0, 0.02, -0.3, 0.5), (3.0, 2.0, 0.6, 0.1),
                                                   (4.0, -0.4, 0.3, 0.3), (200.0, 1.5, 0.3, 0.3)])
def test_caps_and_weights(cap, scale, weight, diff):
    b = cases.batch([40, 17], [(0, 50), (30, 20)], seed=2)
    for dtype in DTYPES:
        got, want = maps_case(dtype, 4, 2, 32, 32, 20, b, 2, seed=1, cap=cap, scale=scale, weight=weight, diff=diff)
        # steep scores carry the rounding of their operands into the weights
        close(got, want, dtype, factor=1.5 if scale < 1 else 4.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(4, 2, 32, 32), (4, 1, 64, 128)])
@pytest.mark.parametrize("query", [47, 48, 63, 64, 90, 127])
def test_a_key_of_either_map_at_the_windows_edge(dtype, heads, kv_heads, dim, vdim, query):
    window = 32
    for key in sorted({query - window + 1, query - window, query - window + 2, 0, 15, 16, 31, 32, query - 1, query}):
        if not 0 <= key <= query:
            continue
        for which in (0, 1):
            for b, n_decode in ((cases.batch([query], [], seed=key), 1), (cases.batch([], [(0, query + 1)], seed=key), 0),
                                (cases.batch([], [(query - 1, 2)], seed=key), 0)):
                got, want = maps_case(dtype, heads, kv_heads, dim, vdim, window, b, n_decode, seed=key, mark=(0, query, key, which), cap=20.0)
                close(got[-1], want[-1], dtype, f"key {key} map {which} decode {n_decode}", factor=2)


def test_many_decoding_requests_and_long_contexts():
    b = cases.batch(np.random.default_rng(0).integers(1, 700, 80).tolist(), [], seed=1)
    got, want = maps_case(BF16, 8, 2, 64, 128, 300, b, 80, seed=2)
    close(got, want, BF16, factor=1.5)
    b = cases.batch([], [(500, 300), (0, 260)], seed=1)
    got, want = maps_case(BF16, 8, 2, 64, 128, 333, b, 0, seed=3)
    close(got, want, BF16, factor=1.5)


def test_the_sink_has_no_place_beside_two_maps():
    b = cases.batch([3], [], seed=0)
    layout = K.kv_layout(F32, 2, 1, 8, 8, 2)
    with pytest.raises(RuntimeError, match="sink"):
        K.window_attention(layout, torch.zeros((1, 4, 32), device="cuda"), K.kv_pool(layout, b.num_pages), device_batch(b), window=0, keep_first=0,
                           scale=1.0, sink=torch.zeros(2, device="cuda"), decode=1)


# ---------------------------------------------------------------- windows over latents

@pytest.mark.parametrize("heads,rank,rot", [(12, 128, 24), (5, 36, 12), (40, 21, 6), (20, 288, 32), (32, 512, 64), (3, 600, 40)])
@pytest.mark.parametrize("window", [1, 24, 64, 100])
def test_latent_window(heads, rank, rot, window):
    b = cases.batch([0, 95, 128, 31, 63, 64], [(0, 70), (50, 41), (33, 2), (0, 1), (112, 16)], seed=rank)
    for dtype in DTYPES:
        got, want = latent_case(dtype, heads, rank, rot, b, 6, seed=rank, window=window)
        close(got, want, dtype, f"{dtype}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("query", [31, 63, 64, 90, 127, 200])
def test_a_latent_key_at_the_windows_edge(dtype, query):
    window = 41
    for key in sorted({0, query - window - 1, query - window, query - window + 1, query - window + 2, query - 1, query}):
        if not 0 <= key <= query:
            continue
        for b, n_decode in ((cases.batch([query], [], seed=key), 1), (cases.batch([], [(0, query + 1)], seed=key), 0),
                            (cases.batch([], [(query - 1, 2)], seed=key), 0)):
            got, want = latent_case(dtype, 6, 48, 8, b, n_decode, seed=key, mark=[(0, query, key)], window=window)
            close(got[-1:], want[-1:], dtype, f"key {key} decode {n_decode}")


# ---------------------------------------------------------------- experts in groups, and one that every token has

@pytest.mark.parametrize("T,experts,groups,keep,top,always", [(1, 6, 3, 2, 3, 1), (37, 8, 4, 1, 2, 0), (130, 64, 8, 3, 8, 2), (300, 12, 12, 5, 5, 1),
                                                              (65, 4, 1, 1, 2, 3), (40, 1000, 250, 20, 60, 4), (700, 130, 2, 1, 4, 1), (9, 1, 1, 1, 1, 1)])
def test_routing_in_groups(T, experts, groups, keep, top, always):
    rng = np.random.default_rng(T)
    ld = (experts + 1 + 7) // 8 * 8
    z = (rng.standard_normal((2, T, ld)) * 1.5).astype(np.float32)
    r, t = K.route(dev(z), experts, experts, top, None, 1.0, 64, groups=groups, keep_groups=keep, always=always)
    zs = z.astype(np.float64).sum(0)
    s = S.softmax(zs[:, :experts])
    chosen = S.grouped_choice(s, top, groups, keep)
    weights = np.concatenate([np.take_along_axis(s, chosen, 1)] + [S.sigmoid(zs[:, experts:experts + 1])] * always, axis=1)
    behind = np.tile(np.arange(experts, experts + always), (T, 1))
    check_routing(t, T, top + always, experts + always, 64, np.concatenate([chosen, behind], axis=1))
    close(t["weight"].reshape(T, top + always), weights, F32)


@pytest.mark.parametrize("T,W,ff,experts,always", [(1, 40, 24, 4, 1), (33, 104, 72, 6, 2), (260, 136, 256, 3, 1), (150, 512, 128, 40, 1)])
def test_squared_relu_experts_and_the_shared_one(T, W, ff, experts, always):
    rng = np.random.default_rng(T)
    top, total = 2, experts + always
    z = rng.standard_normal((1, T, (experts + 1 + 7) // 8 * 8)).astype(np.float32)
    h, x = rng.standard_normal((T, W)), rng.standard_normal((T, W))
    up, down = rng.standard_normal((total, ff, W)) / np.sqrt(W), rng.standard_normal((total, W, ff)) / np.sqrt(ff)
    for dtype in DTYPES:
        per, n = top + always, T * (top + always)
        tile = K.lib().nf_grouped_tile_rows(K.F32 if dtype == F32 else K.BF16, n, total)
        r, _ = K.route(dev(z), experts, experts, top, None, 1.0, tile, always=always)
        s = S.softmax(z[0, :, :experts].astype(np.float64))
        chosen, gate = S.grouped_choice(s, top, 1, 1), S.sigmoid(z[0, :, experts].astype(np.float64))
        dh = dev(h, dtype)
        mid, out = torch.full((n, ff), 9.0, dtype=dtype, device="cuda"), torch.full((n, W), 9.0, dtype=dtype, device="cuda")
        K.gemm_grouped_experts(dh, dev(up, dtype), mid, r, n, True, K.ACT_SQUARED_RELU)
        K.gemm_grouped_experts(mid, dev(down, dtype), out, r, n, False)
        hr, upr, dnr = rounded(h, dtype), rounded(up, dtype), rounded(down, dtype)
        want = x.astype(np.float32).astype(np.float64)
        run = lambda e, v: dnr[e] @ S.squared_relu(upr[e] @ v)
        for token in range(T):
            y = sum(s[token, e] * run(e, hr[token]) for e in chosen[token])
            want[token] += 0.6 * (y + sum(gate[token] * run(e, hr[token]) for e in range(experts, total)))
        dx, act = dev(x, F32), torch.full((T, W), 7.0, dtype=dtype, device="cuda")
        K.mixture_rows(out, r, per, dh, dx, act, W, y_scale=0.6)
        close(dx, want, dtype)
        close(act, want, dtype)


@pytest.mark.parametrize("M,N,Kd", [(1, 8, 8), (64, 264, 1024), (130, 136, 2048), (700, 384, 264)])
def test_products_with_gelu(M, N, Kd):
    rng = np.random.default_rng(M)
    a, b = rng.standard_normal((M, Kd)), rng.standard_normal((N, Kd)) / np.sqrt(Kd)
    ws = torch.empty(1 << 22, dtype=torch.float32, device="cuda")
    for dtype in DTYPES:
        want = S.gelu_erf(rounded(a, dtype) @ rounded(b, dtype).T)
        close(K.gemm_nk(dev(a, dtype), dev(b, dtype), act=K.ACT_GELU, workspace=ws), want, dtype)


@pytest.mark.parametrize("width,ld", [(104, 104), (51, 56), (2050, 2056)])
def test_scaled_sublayers(width, ld):
    rng = np.random.default_rng(width)
    T, eps = 13, 1e-3
    x, y, w = rng.standard_normal((T, width)), rng.standard_normal((2, T, width)), 1.0 + rng.standard_normal(width)
    vec = lambda a: dev(padded(a, ld), F32)
    want = x.astype(np.float32) + 0.35 * y.astype(np.float32).astype(np.float64).sum(0)
    for dtype in DTYPES:
        dx, act = vec(x), torch.full((T, ld), 7.0, dtype=dtype, device="cuda")
        K.residual_rows(vec(y), dx, act, width, None, K.norm(K.NORM_RMS, vec(w), None, eps), y_scale=0.35)
        close(dx[:, :width], want, F32)
        close(act[:, :width], S.rms_norm(want, eps, w), dtype)


def test_capped_scores_of_one_map_beside_a_sink():
    """The cap of plain attention, with kept first positions."""
    b = cases.batch([95, 31], [(0, 70), (50, 41)], seed=3)
    for dtype in DTYPES:
        for shape in ((4, 2, 64, 64), (6, 2, 32, 48)):
            got, want = attention_case(dtype, *shape, 24, 5, b, 2, seed=9, softcap=0.8)
            close(got, want, dtype)
