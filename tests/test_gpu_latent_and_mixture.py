"""Operators of layer-stack models with latent attention, a mixture of experts, layer norms and token inputs, each alone
through the C ABI against the plain float64 statement of its mechanism, in fp32 and in bf16."""
import numpy as np
import pytest

torch = pytest.importorskip("torch")
pytestmark = pytest.mark.gpu

from nanoflow_amd import kernels as K  # noqa: E402
from oracle import stack_oracle as S  # noqa: E402

import stack_cases as cases  # noqa: E402
from test_gpu_stack_kernels import BF16, DTYPES, F32, attention_case, close, dev, device_batch, host, rounded, table_of  # noqa: E402


@pytest.fixture(scope="module", autouse=True)
def _gpu():
    assert torch.cuda.is_available()
    K.lib()


def padded(a, ld):
    return np.pad(a, [(0, 0)] * (a.ndim - 1) + [(0, ld - a.shape[-1])])


# ---------------------------------------------------------------- rows

@pytest.mark.parametrize("width,ld", [(104, 104), (51, 56), (1, 8), (2050, 2056), (9001, 9008)])
def test_layer_norms_after_a_sublayer(width, ld):
    rng = np.random.default_rng(width)
    T, eps = 19, 1e-3
    w, b, nw = (rng.standard_normal(width) for _ in range(3))
    x, y = rng.standard_normal((T, width)) + 3, rng.standard_normal((2, T, width))
    vec = lambda a: dev(padded(a, ld), F32)
    layer = K.norm(K.NORM_LAYER, vec(w), vec(b), eps)
    sums = y.astype(np.float32).astype(np.float64).sum(0)
    for dtype in DTYPES:
        for rms_first in (False, True):
            dx, act = vec(x), torch.full((T, ld), 7.0, dtype=dtype, device="cuda")
            K.residual_rows(vec(y), dx, act, width, K.norm(K.NORM_RMS, vec(nw), None, eps) if rms_first else None, layer)
            want = x.astype(np.float32) + (S.rms_norm(sums, eps, nw) if rms_first else sums)
            close(dx[:, :width], want, F32)
            close(act[:, :width], S.layer_norm(want, eps, w, b), dtype, factor=2)
            assert not host(act[:, width:]).any() and not host(dx[:, width:]).any()
        index = np.array([5, 0, 18, 5], np.int32)
        for i in (None, index):
            got = K.norm_rows(vec(x), None if i is None else dev(i), layer, width, dtype)
            close(got[:, :width], S.layer_norm(x[slice(None) if i is None else i], eps, w, b), dtype, factor=2)
            assert not host(got[:, width:]).any()


@pytest.mark.parametrize("width,o_ld,g_ld", [(96, 96, 104), (70, 72, 70), (13, 13, 15), (4096, 4096, 4096)])
def test_gated_norm(width, o_ld, g_ld):
    rng = np.random.default_rng(width)
    T, eps = 9, 1e-4
    o, g, w = rng.standard_normal((T, o_ld)), rng.standard_normal((T, g_ld)) * 2, rng.standard_normal(width)
    for dtype in DTYPES:
        t = dev(o, dtype)
        K.gated_norm_rows(t, dev(g, dtype), dev(padded(w, (width + 7) // 8 * 8), F32), width, eps)
        want = S.rms_norm(rounded(o, dtype)[:, :width], eps, w) * S.sigmoid(rounded(g, dtype)[:, :width])
        close(t[:, :width], want, dtype)
        np.testing.assert_array_equal(host(t[:, width:]), rounded(o, dtype)[:, width:])


@pytest.mark.parametrize("dim,cols,layers,index", [(20, 24, 3, 2), (8, 8, 1, 0), (5, 8, 4, 1), (256, 256, 2, 1)])
def test_token_gate(dim, cols, layers, index):
    rng = np.random.default_rng(dim)
    T = 21
    z, table, tok = rng.standard_normal((3, T, cols)), rng.standard_normal((11, (dim * layers + 7) // 8 * 8)), rng.integers(0, 11, T).astype(np.int32)
    for dtype in DTYPES:
        got = K.token_gate_rows(dev(z, F32), dev(tok), dev(table, dtype), index * dim, dim)
        want = S.gelu_tanh(z.sum(0)[:, :dim]) * rounded(table, dtype)[tok, index * dim:(index + 1) * dim]
        close(got[:, :dim], want, dtype)
        assert not host(got[:, dim:]).any()


# ---------------------------------------------------------------- mixture

def check_routing(t, T, top, experts, tile_rows, chosen):
    choice, place, row_of = (host(t[k]).astype(int) for k in ("choice", "place", "row_of"))
    choice, place = choice.reshape(T, top), place.reshape(T, top)
    np.testing.assert_array_equal(choice, chosen)
    offsets = host(t["offsets"]).astype(int)
    counts = np.bincount(choice[choice < experts], minlength=experts)
    np.testing.assert_array_equal(np.diff(offsets), counts)
    assert offsets[0] == 0 and (place[choice >= experts] == -1).all()
    used = place[choice < experts]
    assert sorted(used.tolist()) == list(range(counts.sum()))                 # every sorted row once
    for token, k in zip(*np.nonzero(choice < experts)):
        e = choice[token, k]
        assert offsets[e] <= place[token, k] < offsets[e + 1] and row_of[place[token, k]] == token
    n = int(host(t["n_tiles"])[0])
    tiles = list(zip(host(t["tile_group"]).astype(int)[:n].tolist(), host(t["tile_row"]).astype(int)[:n].tolist()))
    assert tiles == [(e, r) for e in range(experts) for r in range(0, counts[e], tile_rows)]


@pytest.mark.parametrize("T,experts,identity,top", [(1, 5, 2, 3), (37, 5, 0, 5), (130, 64, 32, 8), (300, 3, 1, 1), (65, 1, 0, 1), (40, 1000, 24, 60), (700, 2, 7, 4)])
def test_routing(T, experts, identity, top):
    rng = np.random.default_rng(T)
    n = experts + identity
    ld = (n + 7) // 8 * 8
    z, corr = (rng.standard_normal((2, T, ld)) * 1.5).astype(np.float32), rng.standard_normal(n).astype(np.float32) * 0.1
    r, t = K.route(dev(z), n, experts, top, dev(corr), 2.5, 64)
    chosen, w = S.route(z.astype(np.float64).sum(0)[:, :n], corr, top, 2.5)
    check_routing(t, T, top, experts, 64, chosen)
    close(t["weight"].reshape(T, top), w, F32)


def test_equal_scores_choose_the_smaller_index():
    z = torch.zeros((1, 6, 136), dtype=F32, device="cuda")
    r, t = K.route(z, 130, 129, 4, torch.zeros(130, dtype=F32, device="cuda"), 1.0, 64)
    assert host(t["choice"]).astype(int).reshape(6, 4).tolist() == [[0, 1, 2, 3]] * 6
    corr = torch.zeros(130, dtype=F32, device="cuda")
    corr[[129, 70, 6]] = 1.0
    r, t = K.route(z, 130, 129, 4, corr, 1.0, 64)
    assert host(t["choice"]).astype(int).reshape(6, 4).tolist() == [[6, 70, 129, 0]] * 6


@pytest.mark.parametrize("T,W,ff,experts,identity,top", [(1, 40, 24, 4, 2, 2), (33, 104, 72, 5, 2, 3), (260, 136, 256, 3, 0, 2), (600, 64, 520, 2, 3, 4),
                                                         (150, 512, 128, 40, 5, 8), (70, 48, 8, 1, 0, 1)])
def test_experts_and_their_sum(T, W, ff, experts, identity, top):
    """Routing, gathered rows through both products, the weighted sum with identity experts, the norm after it."""
    rng = np.random.default_rng(T)
    n, ld = experts + identity, (W + 7) // 8 * 8
    ldn = (n + 7) // 8 * 8
    z = rng.standard_normal((1, T, ldn)).astype(np.float32)
    if experts > 2:
        z[:, :, 1] = -30.0                                                    # an expert no token asks for
    h, x = rng.standard_normal((T, W)), rng.standard_normal((T, W))
    up, down = rng.standard_normal((experts, ff, W)) / np.sqrt(W), rng.standard_normal((experts, W, ff)) / np.sqrt(ff)
    w, b = rng.standard_normal(W), rng.standard_normal(W)
    for dtype in DTYPES:
        tile = K.lib().nf_grouped_tile_rows(K.F32 if dtype == F32 else K.BF16, T * top, experts)
        r, t = K.route(dev(z), n, experts, top, torch.zeros(n, dtype=F32, device="cuda"), 1.5, tile)
        chosen, weight = S.route(z[0, :, :n].astype(np.float64), np.zeros(n), top, 1.5)
        check_routing(t, T, top, experts, tile, chosen)
        dh = dev(padded(h, ld), dtype)
        mid, out = torch.full((T * top, ff), 9.0, dtype=dtype, device="cuda"), torch.full((T * top, ld), 9.0, dtype=dtype, device="cuda")
        K.gemm_grouped_experts(dh, dev(padded(up, ld), dtype), mid, r, T * top, True, K.ACT_GELU)
        dn = np.zeros((experts, ld, ff))
        dn[:, :W] = down
        K.gemm_grouped_experts(mid, dev(dn, dtype), out, r, T * top, False)
        hr, upr, dnr = rounded(h, dtype), rounded(up, dtype), rounded(down, dtype)
        want = x.astype(np.float32).astype(np.float64)
        for token in range(T):
            for e, wt in zip(chosen[token], weight[token]):
                want[token] += wt * (hr[token] if e >= experts else dnr[e] @ S.gelu_erf(upr[e] @ hr[token]))
        dx, act = dev(padded(x, ld), F32), torch.full((T, ld), 7.0, dtype=dtype, device="cuda")
        vec = lambda a: dev(padded(a, ld), F32)
        K.mixture_rows(out, r, top, dh, dx, act, W, K.norm(K.NORM_LAYER, vec(w), vec(b), 1e-4))
        close(dx[:, :W], want, dtype)
        close(act[:, :W], S.layer_norm(want, 1e-4, w, b), dtype, factor=2)
        # in place: the identity experts' rows and what is left for the next sublayer are one buffer
        dx2 = dev(padded(x, ld), F32)
        K.mixture_rows(out, r, top, dh, dx2, dh, W)
        np.testing.assert_array_equal(host(dx2), host(dx))


@pytest.mark.parametrize("T,heads,N,Kd", [(1, 3, 24, 16), (70, 5, 136, 40), (300, 2, 520, 128), (513, 4, 64, 72), (2, 40, 8, 8)])
def test_products_per_head(T, heads, N, Kd):
    rng = np.random.default_rng(T)
    gap_a, gap_d = Kd + 8, N + 16
    a, b = rng.standard_normal((T, heads * gap_a)), rng.standard_normal((heads, N, Kd)) / np.sqrt(Kd)
    for dtype in DTYPES:
        d = torch.full((T, heads * gap_d), 3.0, dtype=dtype, device="cuda")
        K.gemm_grouped_heads(dev(a, dtype), dev(b, dtype), d, gap_a, gap_d)
        want = np.full((T, heads, gap_d), 3.0)
        want[:, :, :N] = np.einsum("thk,hnk->thn", rounded(a, dtype).reshape(T, heads, gap_a)[:, :, :Kd], rounded(b, dtype))
        close(d, want.reshape(T, -1), dtype)                                  # and nothing beside the heads' columns


# ---------------------------------------------------------------- attention with a gate and a query temperature

@pytest.mark.parametrize("heads,kv_heads,dim,vdim,every", [(4, 2, 64, 64, 16), (6, 1, 24, 40, 7), (3, 3, 18, 10, 1), (2, 1, 160, 256, 1000)])
def test_query_temperature(heads, kv_heads, dim, vdim, every):
    rng = np.random.default_rng(dim)
    b = cases.batch([15, 16, 47], [(0, 37), (every, 3)], seed=dim)
    cols = heads * dim + kv_heads * (dim + vdim)
    proj = rng.standard_normal((b.tokens, cols))
    for dtype in DTYPES:
        layout = K.kv_layout(dtype, heads, kv_heads, dim, vdim)
        d = device_batch(b)
        pools = [K.kv_pool(layout, b.num_pages) for _ in range(2)]
        qs = [K.qkv_append(layout, dev(proj, dtype), (0, heads * dim, (heads + kv_heads) * dim), None, None, 1e-5, K.rotation(), pool, d["kv_indptr"],
                           d["kv_indices"], d["rev_input_indptr"], d["positions"], temp) for pool, temp in zip(pools, ((0.7, every), None))]
        f = S.query_temperature(b.per_token_offset, 0.7, every)[:, None, None]
        close(qs[0][:, :, :dim], rounded(proj, dtype)[:, :heads * dim].reshape(-1, heads, dim) * f, dtype)
        np.testing.assert_array_equal(host(pools[0]), host(pools[1]))          # keys and values have none


@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(4, 2, 64, 64), (5, 1, 18, 10), (20, 1, 16, 16), (3, 3, 160, 96)])
def test_gate_per_head(heads, kv_heads, dim, vdim):
    b = cases.batch([0, 95, 31], [(0, 70), (50, 41), (33, 2)], seed=dim)
    for dtype in DTYPES:
        gate = np.random.default_rng(dim).standard_normal((b.tokens, heads + 3)) * 3
        got, want = attention_case(dtype, heads, kv_heads, dim, vdim, 0, 0, b, 3, seed=dim, gate=gate)
        want = want.reshape(b.tokens, heads, vdim) * S.sigmoid(rounded(gate, dtype)[:, :heads, None])
        close(got, want.reshape(b.tokens, -1), dtype)


# ---------------------------------------------------------------- latent attention

def latent_case(dtype, heads, rank, rot, b, n_decode, seed=0, mark=None, scale=None, workspace=True, window=0):
    """Histories and the batch through append and attention; the plain result for the batch's rows.  mark: (request, query
    position, key position): that key is made to stand out for that query."""
    rng = np.random.default_rng(seed)
    scale = (rank + rot) ** -0.5 if scale is None else scale
    layout = K.latent_layout(dtype, heads, rank, rot)
    width = heads * rot + rank + rot
    ld, weight = (width + 7) // 8 * 8, rng.standard_normal(rank)
    full = [rng.standard_normal((int(n), ld)) for n in b.kv_len]
    queries = [rng.standard_normal((int(n), heads, rank)) for n in b.kv_len]
    plain = []
    for r in range(b.req_num):
        v, pos = rounded(full[r], dtype), np.arange(len(full[r]))
        lat = S.rms_norm(v[:, heads * rot:heads * rot + rank], 1e-5, weight)
        turn = lambda x: S.rotate(x, pos, rot, 60.0, True)
        plain.append((turn(v[:, :heads * rot].reshape(len(v), heads, rot)), lat, turn(v[:, None, heads * rot + rank:width])[:, 0]))
    for r, p, j in mark or []:
        lat = plain[r][1][j]
        queries[r][p] = lat * (12.0 / scale / (lat @ lat))
    table = table_of(int(b.kv_len.max()) + 1, rot, 60.0) if rot else None
    pool = K.latent_pool(layout, b.num_pages)
    pool += 3.0                                                               # what is behind a sequence is not looked at

    def append(batch, rows, qs):
        T = sum(len(r) for r in rows)
        q = torch.full((T, heads, layout.row_ld), 5.0, dtype=dtype, device="cuda")
        q[:, :, :layout.rank_pad] = 0
        q[:, :, :rank] = dev(np.concatenate(qs), dtype)
        K.latent_append(layout, dev(np.concatenate(rows), dtype), (0, heads * rot), dev(padded(weight, layout.rank_pad), F32), 1e-5,
                        K.rotation(table, rot, True), q, pool, device_batch(batch))
        return q

    h, reqs = cases.history_batch(b)
    if h is not None:
        lens = np.diff(h.input_indptr)
        append(h, [full[r][:n] for r, n in zip(reqs, lens)], [queries[r][:n] for r, n in zip(reqs, lens)])
    lens = np.diff(b.input_indptr)
    q = append(b, [full[r][len(full[r]) - n:] for r, n in enumerate(lens)], [queries[r][len(full[r]) - n:] for r, n in enumerate(lens)])
    assert not host(q[:, :, layout.rank_pad + rot:]).any()
    got = K.latent_attention(layout, q, pool, device_batch(b), scale=scale, decode=n_decode, workspace=workspace, window=window)
    want = []
    for r, n in enumerate(lens):
        qr, lat, kr = plain[r]
        T = len(lat)
        qq = np.concatenate([rounded(queries[r], dtype), qr], -1)
        keys = np.concatenate([lat, kr], -1)
        o = S.sink_attention(qq, keys[:, None], lat[:, None], S.window_mask(T, window or T + 1, 0), scale, None)
        want.append(o[T - n:])
    assert not host(got[:, :, rank:]).any()
    return got[:, :, :rank].contiguous(), np.concatenate(want)


@pytest.mark.parametrize("heads,rank,rot", [(12, 128, 24), (1, 64, 64), (5, 36, 12), (40, 21, 6), (32, 192, 0), (17, 256, 64), (20, 288, 32), (32, 512, 64),
                                            (64, 40, 8), (3, 600, 40), (100, 8, 2)])
def test_latent_attention(heads, rank, rot):
    b = cases.batch([0, 95, 128, 31, 63, 64], [(0, 70), (50, 41), (33, 2), (0, 1), (112, 16)], seed=rank)
    for dtype in DTYPES:
        got, want = latent_case(dtype, heads, rank, rot, b, 6, seed=rank)
        close(got, want, dtype, f"{dtype}")


def test_latent_attention_without_room_for_splits_and_with_many_requests():
    b = cases.batch(np.random.default_rng(0).integers(1, 500, 70).tolist(), [], seed=1)
    for heads, workspace in ((8, True), (24, True), (40, True), (24, False)):
        got, want = latent_case(BF16, heads, 64, 16, b, 70, seed=2, workspace=workspace)
        close(got, want, BF16, f"{heads} heads")
    b = cases.batch([700], [(600, 90)], seed=3)
    for workspace in (True, False):
        got, want = latent_case(BF16, 24, 64, 16, b, 1, seed=2, workspace=workspace)
        close(got, want, BF16)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("query", [15, 16, 31, 63, 64, 90, 127, 128, 200])
def test_a_latent_key_far_back_is_found(dtype, query):
    """One key scores far above the others: the first one, the query's own, at the borders of pages and tiles; in a prompt, cut
    before the query, and decoded."""
    for key in sorted({0, 1, 15, 16, 31, 32, 63, 64, query - 1, query}):
        if key > query:
            continue
        for b, n_decode in ((cases.batch([query], [], seed=key), 1), (cases.batch([], [(0, query + 1)], seed=key), 0),
                            (cases.batch([], [(query - 1, 2)], seed=key), 0)):
            got, want = latent_case(dtype, 6, 48, 8, b, n_decode, seed=key, mark=[(0, query, key)])
            close(got[-1:], want[-1:], dtype, f"key {key} decode {n_decode}")


@pytest.mark.parametrize("scale", [0.0, -0.2])
def test_latent_scales_that_are_not_positive(scale):
    b = cases.batch([40], [(0, 50)], seed=2)
    for dtype in DTYPES:
        got, want = latent_case(dtype, 4, 32, 8, b, 1, seed=1, scale=scale)
        close(got, want, dtype)


@pytest.mark.parametrize("heads,dim,vdim,rank,rot", [(4, 16, 24, 36, 12), (3, 10, 9, 21, 6), (2, 128, 128, 64, 64), (6, 48, 72, 96, 24), (5, 32, 16, 24, 0)])
def test_latents_written_out_attend_like_the_heads_they_stand_for(heads, dim, vdim, rank, rot):
    """Prompts beside decode rows, histories in the cache: gather, product, pack and the queries' own form, through the attention over
    pages, against latent attention as it is defined."""
    rng = np.random.default_rng(rank)
    b = cases.batch([37, 5], [(0, 70), (50, 41), (33, 2), (0, 1), (112, 16)], seed=rank)
    p8 = lambda n: (n + 7) // 8 * 8
    dp, vp, rp, scale = p8(dim), p8(vdim), p8(rank), (dim + rot) ** -0.5
    uk, uv, weight = rng.standard_normal((heads, dim, rank)) / np.sqrt(rank), rng.standard_normal((heads, vdim, rank)) / np.sqrt(rank), rng.standard_normal(rank)
    q_col = heads * dp
    kv_col = q_col + heads * rot
    ld = p8(kv_col + rank + rot)
    w = np.zeros((heads * (dp + vp), rp))
    for h in range(heads):
        w[h * dp:h * dp + dim, :rank] = uk[h]
        w[heads * dp + h * vp:heads * dp + h * vp + vdim, :rank] = uv[h]
    table = table_of(int(b.kv_len.max()) + 1, rot, 60.0) if rot else None
    turn = K.rotation(table, rot, True)
    for dtype in DTYPES:
        layout = K.latent_layout(dtype, heads, rank, rot)
        full = []
        for n in b.kv_len:
            x = rng.standard_normal((int(n), ld))
            x[:, :q_col].reshape(len(x), heads, dp)[:, :, dim:] = 0
            full.append(x)
        pool = K.latent_pool(layout, b.num_pages)
        pool += 3.0

        def append(batch, rows):
            q = torch.zeros((sum(len(r) for r in rows), heads, layout.row_ld), dtype=dtype, device="cuda")
            proj = dev(np.concatenate(rows), dtype)
            K.latent_append(layout, proj, (q_col, kv_col), dev(padded(weight, rp), F32), 1e-5, turn, q, pool, device_batch(batch))
            return proj

        h, reqs = cases.history_batch(b)
        append(h, [full[r][:n] for r, n in zip(reqs, np.diff(h.input_indptr))])
        lens = np.diff(b.input_indptr)
        proj = append(b, [full[r][len(full[r]) - n:] for r, n in enumerate(lens)])
        d = device_batch(b)
        n_pages = int(b.kv_indptr[-1] - b.kv_indptr[2])
        kv, pages, ids = K.latent_expand(layout, dp, vp, dev(w, dtype), pool, d, 2, b.req_num, n_pages + 3)
        q = K.latent_queries(kv, dp, proj, q_col, rot, turn, d["positions"], 2, b.tokens - 2)
        out = K.window_attention(kv, q, pages, {**d, "kv_indices": ids}, window=0, keep_first=0, scale=scale, decode=0)
        got = host(out).reshape(b.tokens, heads, vp)[2:]
        want = []
        for r in range(2, b.req_num):
            v, pos, n = rounded(full[r], dtype), np.arange(len(full[r])), lens[r]
            lat = S.rms_norm(v[:, kv_col:kv_col + rank], 1e-5, weight)
            kr = S.rotate(v[:, None, kv_col + rank:kv_col + rank + rot], pos, rot, 60.0, True)[:, 0]
            qr = S.rotate(v[:, q_col:kv_col].reshape(len(v), heads, rot), pos, rot, 60.0, True)
            o = S.latent_attention(v[:, :q_col].reshape(len(v), heads, dp)[:, :, :dim], qr, lat, kr, rounded(uk, dtype), rounded(uv, dtype), scale)
            want.append(o[len(v) - n:])
        close(got[:, :, :vdim], np.concatenate(want), dtype, f"{dtype}", factor=2)
        assert not got[:, :, vdim:].any()
