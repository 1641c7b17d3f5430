"""Operators of layer-stack models with attention in chunks, normed and turned values, sigmoid routing, clamped gated experts and
what a pass over layers starts with, each alone through the C ABI against the plain float64 statement of its mechanism, in fp32
and in bf16; whole models whose layers are passed several times."""
import numpy as np
import pytest

torch = pytest.importorskip("torch")
pytestmark = pytest.mark.gpu

from nanoflow_amd import engine, kernels as K, pllm_python as P  # noqa: E402
from oracle import stack_oracle as S  # noqa: E402

import stack_cases as cases  # noqa: E402
from test_gpu_latent_and_mixture import check_routing, padded  # noqa: E402
from test_gpu_stack_kernels import BF16, DTYPES, F32, close, dev, device_batch, host, rounded, table_of  # noqa: E402


@pytest.fixture(scope="module", autouse=True)
def _gpu():
    assert torch.cuda.is_available()
    K.lib()


# ---------------------------------------------------------------- values: norm, rotation, append

SIZES = [(4, 2, 64, 128), (6, 2, 24, 40), (3, 1, 18, 10), (1, 1, 8, 2), (5, 5, 96, 96), (2, 1, 160, 256), (8, 4, 128, 64)]


@pytest.mark.parametrize("heads,kv_heads,dim,vdim", SIZES)
@pytest.mark.parametrize("norm,turned", [(True, True), (True, False), (False, True)])
def test_values_are_normed_and_turned_where_they_are_cached(heads, kv_heads, dim, vdim, norm, turned):
    """Few rows, and more than a thousand, which take another way to the cache."""
    rng = np.random.default_rng(vdim)
    rot = dim // 2 // 4 * 4
    cols = heads * dim + kv_heads * (dim + vdim)
    qn, kn = rng.standard_normal(dim), rng.standard_normal(dim)
    tab, vtab = table_of(800, rot, 50.0), table_of(800, vdim, 70.0)
    for b in (cases.batch([40, 3], [(0, 37), (21, 30), (5, 2), (30, 1)], seed=dim), cases.batch([9], [(0, 701), (13, 330), (0, 3)], seed=1)):
        proj = rng.standard_normal((b.tokens, (cols + 7) // 8 * 8))
        proj[::3, (heads + kv_heads) * dim:] *= 0.01          # where eps counts
        d, pos = device_batch(b), b.per_token_offset
        for dtype in DTYPES:
            layout = K.kv_layout(dtype, heads, kv_heads, dim, vdim)
            pool = K.kv_pool(layout, b.num_pages)
            q = K.qkv_append(layout, dev(proj, dtype), (0, heads * dim, (heads + kv_heads) * dim), dev(qn, F32), dev(kn, F32), 1e-3, K.rotation(tab, rot), pool,
                             d["kv_indptr"], d["kv_indices"], d["rev_input_indptr"], d["positions"], value_norm=norm,
                             value_rot=K.rotation(vtab, vdim, True) if turned else None)
            v = rounded(proj, dtype)
            close(q[:, :, :dim], S.rotate(S.rms_norm(v[:, :heads * dim].reshape(-1, heads, dim), 1e-3, qn), pos, rot, 50.0, False), dtype)
            val = v[:, (heads + kv_heads) * dim:cols].reshape(-1, kv_heads, vdim)
            val = S.rms_norm(val, 1e-3) if norm else val
            val = S.rotate(val, pos, vdim, 70.0, True) if turned else val
            held, split = host(pool), kv_heads * 16 * layout.k_pad
            pk = held[:, :split].reshape(-1, kv_heads, 16, layout.k_pad)
            pv = held[:, split:].reshape(-1, kv_heads, layout.v_pad, 16)
            page = b.kv_indices[b.kv_indptr[b.rev_input_indptr] + pos // 16]
            close(pv[page, :, :, pos % 16][:, :, :vdim], val, dtype)
            key = v[:, heads * dim:(heads + kv_heads) * dim].reshape(-1, kv_heads, dim)
            close(pk[page, :, pos % 16][:, :, :dim], S.rotate(S.rms_norm(key, 1e-3, kn), pos, rot, 50.0, False), dtype)
            touched = np.zeros((b.num_pages, 16), bool)
            touched[page, pos % 16] = True
            assert not pv.transpose(0, 3, 1, 2)[~touched].any() and not pv[:, :, vdim:].any()


# ---------------------------------------------------------------- attention in chunks, outputs turned back

def chunk_case(dtype, heads, kv_heads, dim, vdim, chunk, b, n_decode, seed=0, mark=None, turned=True, sink_scale=1.0, window=0, keep=0, gate=False,
               head_norm=False, base=60.0):
    """Histories and the batch through append and attention; the plain result for the batch's rows.  mark: (request, query, key): that key
    is made to stand out for that query."""
    rng = np.random.default_rng(seed)
    scale = dim ** -0.5
    qn, kn = heads * dim, kv_heads * dim
    cols = qn + kn + kv_heads * vdim
    full = [rng.standard_normal((int(n), (cols + 7) // 8 * 8)) for n in b.kv_len]
    if mark:
        r, p, j = mark
        key = full[r][j, qn:qn + kn].reshape(kv_heads, dim)
        key *= 3.0
        full[r][p, :qn] = np.repeat(key, heads // kv_heads, 0).ravel() * (14.0 / (9.0 * dim * scale))
    sink = rng.standard_normal(heads) * sink_scale
    layout = K.kv_layout(dtype, heads, kv_heads, dim, vdim)
    pool = K.kv_pool(layout, b.num_pages)
    vrot = K.rotation(table_of(int(max(b.kv_len)) + 1, vdim, base), vdim, True) if turned else None

    def append(batch, rows):
        d = device_batch(batch)
        return K.qkv_append(layout, dev(np.concatenate(rows), dtype), (0, qn, qn + kn), None, None, 1e-5, K.rotation(), pool, d["kv_indptr"],
                            d["kv_indices"], d["rev_input_indptr"], d["positions"], value_norm=True, value_rot=vrot)

    h, reqs = cases.history_batch(b)
    if h is not None:
        append(h, [full[r][:n] for r, n in zip(reqs, np.diff(h.input_indptr))])
    lens = np.diff(b.input_indptr)
    q = append(b, [full[r][len(full[r]) - n:] for r, n in enumerate(lens)])
    g = rng.standard_normal((b.tokens, heads)) * 2 if gate else None
    got = K.window_attention(layout, q, pool, device_batch(b), window=window, keep_first=keep, scale=scale, sink=dev(sink, F32), decode=n_decode, chunk=chunk,
                             out_rot=vrot, out_scale=0.8, gate=None if g is None else dev(g, dtype), head_eps=1e-4 if head_norm else None)
    want = []
    for r, n in enumerate(lens):
        v = rounded(full[r], dtype)
        T = len(v)
        i, j = np.arange(T)[:, None], np.arange(T)[None, :]
        near = (i - j < window) if window else True
        mask = (j <= i) & ((near & ((i // chunk == j // chunk) if chunk else True)) | (j < keep))
        val = S.rms_norm(v[:, qn + kn:cols].reshape(T, kv_heads, vdim), 1e-5)
        pos = np.arange(T)
        val = S.rotate(val, pos, vdim, base, True) if turned else val
        o = S.sink_attention(v[:, :qn].reshape(T, heads, dim), v[:, qn:qn + kn].reshape(T, kv_heads, dim), val, mask, scale, sink)
        o = S.rotate(o, -pos, vdim, base, True) if turned else o
        o = S.rms_norm(o, 1e-4) if head_norm else o
        want.append(0.8 * o[T - n:])
    want = np.concatenate(want)
    if gate:
        want = want * S.sigmoid(rounded(g, dtype))[:, :, None]
    return got, want.reshape(len(want), -1)


@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(4, 2, 64, 64), (6, 2, 32, 48), (5, 1, 18, 10), (20, 1, 128, 128), (3, 3, 192, 128), (2, 1, 160, 256), (7, 1, 96, 80),
                                                     (40, 2, 8, 2)])
@pytest.mark.parametrize("chunk", [24, 1, 64, 0, 200, 37])
def test_attention_in_chunks(heads, kv_heads, dim, vdim, chunk):
    b = cases.batch([0, 95, 128, 31, 63, 64], [(0, 70), (50, 41), (33, 2), (0, 1), (112, 16), (47, 3)], seed=chunk)
    for dtype in DTYPES:
        got, want = chunk_case(dtype, heads, kv_heads, dim, vdim, chunk, b, 6, seed=dim)
        close(got, want, dtype, f"{dtype}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(4, 2, 32, 32), (4, 1, 128, 128)])
@pytest.mark.parametrize("chunk", [32, 40, 104])
def test_a_key_at_the_chunks_edge(dtype, heads, kv_heads, dim, vdim, chunk):
    """Keys just inside and just outside the query's chunk, at the borders of pages and far back in it, for queries at either end of a chunk."""
    for query in (chunk - 1, chunk, chunk + 1, 2 * chunk - 1, 2 * chunk + 17):
        start = query // chunk * chunk
        for key in sorted({0, 15, 16, start - 2, start - 1, start, start + 1, start + 15, start + 16, query - 1, query}):
            if not 0 <= key <= query:
                continue
            for b, n_decode in ((cases.batch([query], [], seed=key), 1), (cases.batch([], [(0, query + 1)], seed=key), 0),
                                (cases.batch([], [(query - 1, 2)], seed=key), 0)):
                got, want = chunk_case(dtype, heads, kv_heads, dim, vdim, chunk, b, n_decode, seed=key, mark=(0, query, key))
                close(got[-1], want[-1], dtype, f"query {query} key {key} decode {n_decode}", factor=2)


@pytest.mark.parametrize("window,keep,gate,head_norm,turned", [(15, 0, False, False, True), (15, 5, True, False, True), (0, 9, False, True, True), (0, 0, True, True, False),
                                                               (50, 3, False, False, False)])
def test_chunks_beside_the_other_forms(window, keep, gate, head_norm, turned):
    b = cases.batch([40, 17, 96], [(0, 50), (30, 45), (63, 2)], seed=2)
    for dtype in DTYPES:
        for shape in ((4, 2, 64, 64), (6, 2, 24, 40)):
            got, want = chunk_case(dtype, *shape, 32, b, 3, seed=3, window=window, keep=keep, gate=gate, head_norm=head_norm, turned=turned)
            close(got, want, dtype, factor=2 if head_norm else 1)


@pytest.mark.parametrize("sink_scale", [0.0, 4.0])
def test_the_sink_counts_once_in_every_chunk(sink_scale):
    """Rows that see one key or a few, where the sink's share is large."""
    b = cases.batch([32, 33, 64, 0], [(32, 2), (0, 40)], seed=5)
    for dtype in DTYPES:
        got, want = chunk_case(dtype, 4, 2, 32, 32, 32, b, 4, seed=6, sink_scale=sink_scale)
        close(got, want, dtype)


def test_many_decoding_requests_and_long_contexts_in_chunks():
    b = cases.batch(np.random.default_rng(0).integers(1, 1500, 80).tolist(), [], seed=1)
    got, want = chunk_case(BF16, 8, 2, 64, 128, 700, b, 80, seed=2)
    close(got, want, BF16)
    b = cases.batch([], [(500, 300), (0, 260), (1300, 5)], seed=1)
    got, want = chunk_case(BF16, 8, 2, 128, 128, 333, b, 0, seed=3)
    close(got, want, BF16)


# ---------------------------------------------------------------- routing by sigmoids, clamped gated experts

@pytest.mark.parametrize("T,experts,top,always", [(1, 6, 3, 1), (37, 8, 2, 0), (130, 64, 8, 2), (300, 12, 1, 1), (65, 4, 4, 3), (40, 1000, 60, 4), (9, 1, 1, 1)])
def test_routing_by_sigmoids(T, experts, top, always):
    rng = np.random.default_rng(T)
    ld = (experts + 7) // 8 * 8                      # no column for a gate
    z = (rng.standard_normal((2, T, ld)) * 1.5).astype(np.float32)
    r, t = K.route(dev(z), experts, experts, top, None, 1.0, 64, always=always, scores=K.SCORES_SIGMOID, always_plain=True)
    chosen, s = S.sigmoid_choice(z.astype(np.float64).sum(0)[:, :experts], top)
    behind = np.tile(np.arange(experts, experts + always), (T, 1))
    check_routing(t, T, top + always, experts + always, 64, np.concatenate([chosen, behind], axis=1))
    weights = np.concatenate([s, np.ones((T, always))], axis=1)
    close(t["weight"].reshape(T, top + always), weights, F32)
    place = host(t["place"]).astype(int).reshape(T, top + always)
    close(host(t["row_weight"])[place], weights, F32)


@pytest.mark.parametrize("T,W,ff,experts,top,always", [(1, 40, 24, 4, 2, 1), (33, 104, 72, 6, 1, 2), (260, 136, 256, 3, 3, 1), (150, 512, 128, 40, 4, 0), (700, 64, 40, 2, 1, 1),
                                                       (300, 264, 136, 2, 2, 1)])
def test_gated_experts_of_weighed_inputs(T, W, ff, experts, top, always):
    """Gate and up side by side in the stacked weights, limits of their own for the experts that every token has."""
    rng = np.random.default_rng(T)
    total, per = experts + always, top + always
    n, eps = T * per, 1e-3
    z = rng.standard_normal((1, T, (experts + 7) // 8 * 8)).astype(np.float32)
    h, x, nw = rng.standard_normal((T, W)), rng.standard_normal((T, W)), rng.standard_normal(W)
    gate, up = (rng.standard_normal((total, ff, W)) / np.sqrt(W) for _ in range(2))
    down = rng.standard_normal((total, W, ff)) / np.sqrt(ff)
    limits = np.where(np.arange(total) < experts, 0.4, 1.1)
    for dtype in DTYPES:
        tile = K.lib().nf_grouped_tile_rows(K.F32 if dtype == F32 else K.BF16, n, total)
        r, _ = K.route(dev(z), experts, experts, top, None, 1.0, tile, always=always, scores=K.SCORES_SIGMOID, always_plain=True)
        chosen, s = S.sigmoid_choice(z[0, :, :experts].astype(np.float64), top)
        mid, out = torch.full((n, ff), 9.0, dtype=dtype, device="cuda"), torch.full((n, W), 9.0, dtype=dtype, device="cuda")
        pairs = np.stack([gate, up], 2).reshape(total, 2 * ff, W)
        K.gemm_grouped_experts(dev(h, dtype), dev(pairs, dtype), mid, r, n, True, K.ACT_GATED, weigh=True, gated=(1.702, 1.0, dev(limits, F32)))
        K.gemm_grouped_experts(mid, dev(down, dtype), out, r, n, False)
        hr, gr, ur, dr = (rounded(a, dtype) for a in (h, gate, up, down))
        y = np.zeros((T, W))
        for token in range(T):
            for e, w in [*zip(chosen[token], s[token]), *((e, 1.0) for e in range(experts, total))]:
                y[token] += S.clamped_expert({"gate": gr[e], "up": ur[e], "down": dr[e]}, "", limits[e], w * hr[token])
        for norm in (False, True):
            dx, act = dev(x, F32), torch.full((T, W), 7.0, dtype=dtype, device="cuda")
            K.mixture_rows(out, r, per, None, dx, act, W, plain=True, y_norm=K.norm(K.NORM_RMS, dev(nw, F32), None, eps) if norm else None)
            want = x.astype(np.float32) + (S.rms_norm(y, eps, nw) if norm else y)
            close(dx, want, dtype, factor=2)
            close(act, want, dtype, factor=2)


def test_a_plain_swiglu_is_a_gated_act_without_limits():
    rng = np.random.default_rng(0)
    T, W, ff = 50, 72, 40
    h, w = rng.standard_normal((T, W)), rng.standard_normal((1, 2 * ff, W)) / np.sqrt(W)
    for dtype in DTYPES:
        tile = K.lib().nf_grouped_tile_rows(K.F32 if dtype == F32 else K.BF16, T, 1)
        r, _ = K.route(torch.zeros((1, T, 8), device="cuda"), 1, 1, 1, None, 1.0, tile)
        d = torch.zeros((T, ff), dtype=dtype, device="cuda")
        K.gemm_grouped_experts(dev(h, dtype), dev(w, dtype), d, r, T, True, K.ACT_GATED)
        p = rounded(h, dtype) @ rounded(w[0], dtype).T
        close(d, (S.silu(p[:, ::2]) * p[:, 1::2])[host(r_rows(r, T)).astype(int)], dtype)


def r_rows(r, n):
    """Tokens of the sorted rows (one expert has them in any order)."""
    import ctypes
    buf = torch.empty(n, dtype=torch.int32, device="cuda")
    torch.cuda.synchronize()
    assert ctypes.CDLL("libamdhip64.so").hipMemcpy(ctypes.c_void_p(buf.data_ptr()), ctypes.c_void_p(r.row_of), ctypes.c_size_t(4 * n), ctypes.c_int(4)) == 0
    return buf


# ---------------------------------------------------------------- rows

@pytest.mark.parametrize("width,ld", [(104, 104), (51, 56), (2050, 2056), (9000, 9000)])
def test_what_a_pass_starts_with(width, ld):
    """After a sublayer's output, and with none: a vector, and rows of a table by token."""
    rng = np.random.default_rng(width)
    T, eps = 23, 1e-3
    x, y, w, add, table = (rng.standard_normal(s) for s in ((T, width), (1, T, width), width, width, (9, width)))
    tok = rng.integers(0, 9, T).astype(np.int32)
    vec = lambda a: dev(padded(a, ld), F32)
    for dtype in DTYPES:
        dtab = dev(padded(table, ld), dtype)
        for sub in (False, True):
            for a, tab in ((True, False), (True, True), (False, True)):
                dx, act = vec(x), torch.full((T, ld), 7.0, dtype=dtype, device="cuda")
                K.residual_rows(vec(y) if sub else None, dx, act, width, K.norm(K.NORM_RMS, vec(w), None, eps) if sub else None,
                                K.norm(K.NORM_RMS, vec(w), None, eps), add=vec(add) if a else None, table=dtab if tab else None, tokens=dev(tok) if tab else None,
                                table_scale=2.5)
                want = x + (S.rms_norm(y[0], eps, w) if sub else 0) + (add if a else 0) + (2.5 * rounded(table, dtype)[tok] if tab else 0)
                close(dx[:, :width], want, F32)
                close(act[:, :width], S.rms_norm(want, eps, w), dtype)
                assert not host(dx[:, width:]).any()
        gx, _ = K.embed_rows(dev(tok), dev(tok), dtab, None, scale=1.7)
        close(gx[:, :width], 1.7 * rounded(table, dtype)[tok], F32)


# ---------------------------------------------------------------- whole models

@pytest.fixture
def llama_again():
    yield
    import os
    P.setModelConfig(os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "nanoflow_amd", "config_all", "llama3-8B.json"))


def logits_of(cfg, bits, tok, cuts, dtype="float32"):
    with engine.StackEngine(cfg, dtype=dtype, global_batch=256, kv_pages=24, state_slots=2, weights=bits) as e:
        r, out, at = e.replay(), [], 0
        for n in cuts:
            out.append(r.step([("a", tok[at:at + n], range(n))], e.vocab)["a"])
            at += n
        r.close()
    return np.concatenate(out)


@pytest.mark.parametrize("loop", [(0, 1, 1), (0, 1, 4), (1, 3, 2), (2, 3, 3), (0, 3, 2), None])
def test_loops_of_any_place_and_number(loop, llama_again):
    """Every pass has its own keys and values: prompts, portions and single tokens, also where the loop starts with the first layer or
    ends with the last."""
    cfg = cases.desalix([(cases.chunked(chunk=24), cases.gated_moe()), (cases.chunked(heads=2, kv_heads=1, dim=16, vdim=8, chunk=9), None),
                         (cases.chunked(chunk=40), cases.gated_moe(3, 1, 16, 0.5, None))], loop=loop, width=64, vocab=50)
    bits, t = cases.tensors(cfg)
    tok = np.random.default_rng(1).integers(0, 50, 60)
    want = S.forward(cfg, t, tok)
    scale = np.sqrt((want ** 2).mean())
    for cuts in ([60], [30] + [1] * 30, [2] * 30, [7, 1, 1, 15, 2, 34]):
        assert np.abs(logits_of(cfg, bits, tok, cuts) - want).max() <= 2e-4 * scale, cuts


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_far_key_inside_and_outside_the_chunk(dtype, llama_again):
    """One token's key stands out for a later token, by weights made for it: the answer changes with that token exactly where it is in
    the same chunk."""
    chunk, dim, W, V = 48, 32, 64, 40
    cfg = cases.desalix([(cases.chunked(heads=2, kv_heads=1, dim=dim, vdim=32, chunk=chunk, rot=0, scale=1.0), None)], width=W, vocab=V, scale=3.0)
    rng = np.random.default_rng(2)
    bits, t = cases.tensors(cfg)
    from nanoflow_amd import stack_models
    new = {k: v.copy() for k, v in t.items()}
    # columns 0 and 1 of the embedding mark the asking token 39 and the answering tokens 37 and 38
    new["embed"][:, :3] = 0
    new["embed"][39, 0] = new["embed"][37, 1] = new["embed"][38, 1] = 8.0
    new["l0.mix.q"] *= 0.02
    new["l0.mix.k"] *= 0.02
    for head in range(2):
        new["l0.mix.q"][head * dim, 0] = 30.0
    new["l0.mix.k"][0, 1] = 30.0
    new["l0.mix.q.norm"][:] = 1.0
    new["l0.mix.k.norm"][:] = 1.0
    bits = {k: stack_models.bf16_bits(v) for k, v in new.items()}
    t = {k: stack_models.bits_to_f32(v) for k, v in bits.items()}
    T, query = 140, 100                               # chunk 96 .. 143
    base = rng.integers(0, 37, T)
    base[query] = 39
    for key in (96, 97, 99, 95, 94, 48, 0):
        rows = []
        for answer in (37, 38):
            tok = base.copy()
            tok[key] = answer
            want = S.forward(cfg, t, tok)[query]
            for cuts in ([query + 1], [query, 1], [query - 3, 2, 2]):
                got = logits_of(cfg, bits, tok, cuts, dtype)[query]
                assert np.abs(got - want).max() <= (1e-3 if dtype == "float32" else 0.02) * np.abs(want).max(), (key, cuts)
            rows.append(want)
        differ = np.abs(rows[0] - rows[1]).max() / np.abs(rows[0]).max()
        assert differ > 0.05 if key >= 96 else differ < 1e-9, (key, differ)
