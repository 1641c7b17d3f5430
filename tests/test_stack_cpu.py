"""Layer-stack models without a GPU: the plain implementation against other statements of the same mechanisms,
configurations, state slots in the batch former."""
import ctypes
import json

import numpy as np
import pytest

from nanoflow_amd import pllm_python as P, stack_models
from oracle import stack_oracle as S

import stack_cases as cases


def test_fixed_decay_recurrence_is_a_decayed_sum():
    rng = np.random.default_rng(0)
    q, k, v = rng.standard_normal((9, 2, 5)), rng.standard_normal((9, 2, 5)), rng.standard_normal((9, 2, 3))
    decay = [0.5, 0.9]
    o = S.fixed_decay_recurrence(q, k, v, decay)
    for t in range(9):
        for h in range(2):
            want = sum(decay[h] ** (t - j) * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1))
            np.testing.assert_allclose(o[t, h], want, rtol=1e-12)


def test_bonus_recurrence_is_a_decayed_sum():
    rng = np.random.default_rng(1)
    r, k, v = rng.standard_normal((8, 2, 4)), rng.standard_normal((8, 2, 4)), rng.standard_normal((8, 2, 3))
    w, u = rng.random((8, 2, 4)), rng.standard_normal((2, 4))
    o = S.bonus_recurrence(r, k, v, w, u)
    for t in range(8):
        for h in range(2):
            want = (r[t, h] * u[h] * k[t, h]).sum() * v[t, h]
            for j in range(t):
                keep = np.prod(w[j + 1:t, h], axis=0)
                want = want + (r[t, h] * keep * k[j, h]).sum() * v[j, h]
            np.testing.assert_allclose(o[t, h], want, rtol=1e-12)


@pytest.mark.parametrize("interleaved", [False, True])
def test_rotation_depends_on_distance_only_and_leaves_the_rest(interleaved):
    rng = np.random.default_rng(2)
    a, b = rng.standard_normal((1, 1, 10)), rng.standard_normal((1, 1, 10))
    dots = [(S.rotate(a, [p + 7], 6, 100.0, interleaved) * S.rotate(b, [p], 6, 100.0, interleaved))[..., :6].sum() for p in (0, 3, 50)]
    np.testing.assert_allclose(dots, dots[0], rtol=1e-12)
    np.testing.assert_array_equal(S.rotate(a, [9], 6, 100.0, interleaved)[..., 6:], a[..., 6:])
    np.testing.assert_array_equal(S.rotate(a, [0], 6, 100.0, interleaved), a)


def test_window_mask_edges():
    m = S.window_mask(40, 8, 3)
    assert m[30, 23] and not m[30, 22] and m[30, 2] and not m[30, 3] and not m[30, 31] and m[5, 0]


def test_sink_takes_its_share():
    q = np.zeros((1, 1, 4))
    o = S.sink_attention(q, np.zeros((1, 1, 4)), np.ones((1, 1, 2)), np.ones((1, 1), bool), 1.0, [np.log(3.0)])
    np.testing.assert_allclose(o, 0.25)
    np.testing.assert_allclose(S.sink_attention(q, np.zeros((1, 1, 4)), np.ones((1, 1, 2)), np.ones((1, 1), bool), 1.0, None), 1.0)


def test_layer_norm_and_its_shift_invariance():
    x = np.random.default_rng(0).standard_normal((5, 9)) * 3 + 7
    w, b = np.arange(9) + 1.0, np.linspace(-1, 1, 9)
    y = (S.layer_norm(x, 0.0, w, b) - b) / w
    np.testing.assert_allclose(y.mean(1), 0, atol=1e-12)
    np.testing.assert_allclose(y.std(1), 1, rtol=1e-12)
    np.testing.assert_allclose(S.layer_norm(x + 100, 0.0, w, b), S.layer_norm(x, 0.0, w, b), rtol=1e-9, atol=1e-9)


def test_activations():
    import torch
    z = np.linspace(-6, 6, 101)
    t = torch.from_numpy(z)
    np.testing.assert_allclose(S.gelu_erf(z), torch.nn.functional.gelu(t), atol=1e-12)
    np.testing.assert_allclose(S.gelu_tanh(z), torch.nn.functional.gelu(t, approximate="tanh"), atol=1e-12)


def test_query_temperature_steps_at_block_borders():
    f = S.query_temperature(np.arange(20), 0.5, 4)
    assert np.all(f[:3] == 1) and np.all(f[3:7] == f[3]) and f[3] == 1 + 0.5 * np.log(2) and f[7] == 1 + 0.5 * np.log(3)


def test_latent_attention_is_the_same_multiplied_into_the_latent_space():
    rng = np.random.default_rng(4)
    T, H, d, r, c, e = 12, 3, 5, 4, 7, 6
    q, qr, lat, kr = rng.standard_normal((T, H, d)), rng.standard_normal((T, H, r)), rng.standard_normal((T, c)), rng.standard_normal((T, r))
    uk, uv = rng.standard_normal((H, d, c)), rng.standard_normal((H, e, c))
    want = S.latent_attention(q, qr, lat, kr, uk, uv, 0.4)
    qq = np.concatenate([np.einsum("thd,hdc->thc", q, uk), qr], -1)
    o = S.sink_attention(qq, np.concatenate([lat, kr], -1)[:, None], lat[:, None], S.window_mask(T, T + 1, 0), 0.4, None)
    np.testing.assert_allclose(np.einsum("thc,hec->the", o, uv), want, rtol=1e-9)


def test_routing_chooses_with_the_correction_and_weighs_without_it():
    z = np.log(np.array([[0.1, 0.2, 0.3, 0.4]]))
    chosen, w = S.route(z, np.array([0.5, 0.0, 0.0, 0.0]), 2, 3.0)
    assert chosen.tolist() == [[0, 3]]
    np.testing.assert_allclose(w, [[0.3, 1.2]])


def test_identity_experts_return_their_input():
    t = {"m.router": np.zeros((3, 4)), "m.correction": np.array([0.0, 1.0, 1.0])}
    h = np.random.default_rng(0).standard_normal((5, 4))
    y = S.mixture(t, "m.", {"router": {"experts": 1, "identity": 2, "top": 2, "scale": 1.5}}, h)
    np.testing.assert_allclose(y, h)


def test_a_short_convolution_is_a_causal_filter():
    rng = np.random.default_rng(5)
    u, w = rng.standard_normal((9, 3)), rng.standard_normal((3, 4))
    for c in range(3):
        np.testing.assert_allclose(S.short_conv(u, w)[:, c], np.convolve(u[:, c], w[c, ::-1])[:9], rtol=1e-9, atol=1e-12)


def test_stretched_frequencies_meet_at_both_ends():
    lengths = np.array([10.0, 99.999, 100.001, 200.0, 299.999, 300.001, 5000.0])       # of waves; 300 positions, low 1, high 3
    f = 2 * np.pi / lengths
    g = S.stretched_frequencies(f, 4.0, 1.0, 3.0, 300)
    np.testing.assert_allclose(g[:2], f[:2])
    np.testing.assert_allclose(g[5:], f[5:] / 4)
    np.testing.assert_allclose(g[[2, 4]], [f[2], f[4] / 4], rtol=1e-4)
    np.testing.assert_allclose(g[3], f[3] * (0.25 + 0.75 * 0.25))                       # 1.5 waves: a quarter of the way


def test_rotation_by_angles_is_the_rotation_by_halves():
    x, p = np.random.default_rng(6).standard_normal((7, 2, 11)), np.arange(7)
    angles = p[:, None] * 50.0 ** (-2.0 * np.arange(4) / 8)
    np.testing.assert_allclose(S.rotate_by(x, angles), S.rotate(x, p, 8, 50.0, False), rtol=1e-12)


def test_capped_scores():
    s = np.array([-1e6, -0.01, 0.0, 0.01, 1e6])
    np.testing.assert_allclose(S.capped(s, 5.0), [-5.0, -0.01, 0.0, 0.01, 5.0], rtol=1e-5)
    assert S.capped(s, None) is s


def test_the_difference_of_two_maps():
    """Without the second map it is plain attention, normed; with equal maps a shorter copy of it, which the norm takes back."""
    rng = np.random.default_rng(7)
    q, k, v = rng.standard_normal((8, 4, 2, 5)), rng.standard_normal((8, 2, 2, 5)), rng.standard_normal((8, 2, 3))
    mask = S.window_mask(8, 4, 0)
    plain = S.rms_norm(S.sink_attention(q[:, :, 0], k[:, :, 0], v, mask, 0.4, None), 0.0) * 0.7
    np.testing.assert_allclose(S.differential_attention(q, k, v, mask, 0.4, None, 0.0, 0.3, 0.0), plain, rtol=1e-9)
    q[:, :, 1], k[:, :, 1] = q[:, :, 0], k[:, :, 0]
    np.testing.assert_allclose(S.differential_attention(q, k, v, mask, 0.4, None, 0.6, 0.3, 0.0), plain, rtol=1e-9)
    assert S.map_weight([0.0], [3.0], [1.0], [0.0], 0.3) == 0.3


def test_choice_is_made_in_the_best_groups():
    s = np.array([[0.05, 0.30, 0.20, 0.19, 0.01, 0.25]])          # groups of two: best 0.30, 0.20, 0.25
    assert S.grouped_choice(s, 3, 3, 2).tolist() == [[1, 5, 0]]
    assert S.grouped_choice(s, 3, 3, 3).tolist() == S.grouped_choice(s, 3, 1, 1).tolist() == [[1, 5, 2]]
    assert S.grouped_choice(s, 2, 3, 1).tolist() == [[1, 0]]


def test_latent_window_leaves_out_what_is_behind_it():
    rng = np.random.default_rng(8)
    q, qr, lat, kr = rng.standard_normal((9, 2, 3)), rng.standard_normal((9, 2, 2)), rng.standard_normal((9, 4)), rng.standard_normal((9, 2))
    uk, uv = rng.standard_normal((2, 3, 4)), rng.standard_normal((2, 5, 4))
    o = S.latent_attention(q, qr, lat, kr, uk, uv, 0.4, S.window_mask(9, 3, 0))
    np.testing.assert_allclose(o[8], S.latent_attention(q[6:], qr[6:], lat[6:], kr[6:], uk, uv, 0.4)[2], rtol=1e-9)


def test_chunk_mask_edges():
    m = S.chunk_mask(30, 8)
    assert m[15, 8] and not m[15, 7] and m[16, 16] and not m[16, 15] and not m[16, 17] and m[7, 0]
    assert np.array_equal(S.chunk_mask(30, 1), np.eye(30, dtype=bool)) and np.array_equal(S.chunk_mask(9, None), np.tri(9, dtype=bool))


def test_turned_values_come_back_turned_by_the_distance():
    """A weighted sum of turned values, turned back at the query, is the sum of the values turned by key less query."""
    rng = np.random.default_rng(9)
    v, a = rng.standard_normal((6, 1, 8)), rng.random(6)
    o = S.turn_values((a[:, None, None] * S.turn_values(v, np.arange(6), 40.0)).sum(0, keepdims=True), [5], 40.0, back=True)
    want = sum(a[j] * S.turn_values(v[j:j + 1], [j - 5], 40.0) for j in range(6))
    np.testing.assert_allclose(o, want, rtol=1e-12)
    np.testing.assert_allclose(S.turn_values(v, np.arange(6), 40.0), S.rotate(v, np.arange(6), 8, 40.0, False), rtol=1e-12)


def test_a_clamped_experts_bounds():
    t = {"gate": np.array([[1.0], [1.0]]), "up": np.array([[1.0], [-1.0]]), "down": np.eye(2)}
    sig = lambda z: 1 / (1 + np.exp(-z))
    y = S.clamped_expert(t, "", 2.0, np.array([[1.0], [5.0], [-5.0]]))
    np.testing.assert_allclose(y[0], [sig(1.702) * 2, 0], atol=1e-12)
    np.testing.assert_allclose(y[1], [2 * sig(3.404) * 3, -2 * sig(3.404)])             # both bounded
    np.testing.assert_allclose(y[2], [5 * sig(-8.51), -15 * sig(-8.51)])                # a gate is not bounded from below


def test_weights_go_into_the_experts_and_are_not_shared_out():
    rng = np.random.default_rng(10)
    W, f = 5, 4
    t = {f"m.e{e}.{s}": rng.standard_normal((W, f) if s == "down" else (f, W)) for e in range(3) for s in ("gate", "up", "down")}
    t["m.router"] = np.zeros((3, W))
    t["m.router"][:, 0] = [0.0, 2.0, 1.0]
    h = np.ones((1, W))
    y = S.input_weighted_mixture(t, "m.", {"router": {"top": 2}, "expert": {"limit": 0.5}}, h)
    np.testing.assert_allclose(y, S.clamped_expert(t, "m.e1.", 0.5, h / (1 + np.exp(-2.0))) + S.clamped_expert(t, "m.e2.", 0.5, h / (1 + np.exp(-1.0))), rtol=1e-9)


def test_order_of_looped_layers():
    loop = {"start": 1, "stop": 3, "times": 2}
    assert S.layer_runs(4, loop) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert S.layer_runs(2, None) == [(0, None), (1, None)] and S.layer_runs(1, {"start": 0, "stop": 1, "times": 3}) == [(0, 0), (0, 1), (0, 2)]


@pytest.mark.parametrize("name", ["mixed", "five layers", "two maps", "odd maps", "chunks", "odd chunks"])
def test_a_prefix_does_not_see_what_follows(name):
    cfg = cases.CONFIGS[name]
    _, t = cases.tensors(cfg)
    tokens = np.random.default_rng(3).integers(0, cfg["vocab"], 50)
    whole = S.forward(cfg, t, tokens)
    np.testing.assert_allclose(S.forward(cfg, t, tokens[:31]), whole[:31], rtol=1e-9, atol=1e-9)


def _set(tmp_path, cfg, dtype="bfloat16", pages=8, slots=2):
    p = tmp_path / "config.json"
    p.write_text(json.dumps(cfg))
    P.stackSetConfig(str(p), dtype, 64, pages, slots)


def test_configurations_are_checked(tmp_path):
    try:
        for name, cfg in cases.CONFIGS.items():
            _set(tmp_path, cfg, slots=3)
            assert P.stackStateSlots() == 3 and P.maxPageNum() == 8
        good = cases.CONFIGS["mixed"]
        bad = [({**good, "architecture": "Nosuch"}, "unknown architecture"), ({k: v for k, v in good.items() if k != "width"}, "width"),
               ({**good, "layers": []}, "layers"), (cases.config([cases.parallel(heads=5, kv_heads=2)]), "multiple"),
               (cases.config([cases.retention(heads=3, decay=(0.5, 0.5))]), "decay"),
               (cases.config([cases.retention(rot=17)]), "rotated"), (cases.config([cases.parallel(window=0)]), "mask"),
               (cases.config([cases.retention(dim=300)]), "head sizes"),
               ({**good, "layers": [{**good["layers"][0], "type": "nosuch"}]}, "unknown mixer"),
               ({**good, "layers": [{**good["layers"][0], "mlp": {"kind": "nosuch", "ff": 8}}]}, "feed-forward"),
               (cases.fipuzen([cases.attention(heads=5, kv_heads=2)]), "multiple"), (cases.fipuzen([cases.attention(q_temp=(1.0, 0))]), "temperature"),
               (cases.fipuzen([cases.attention(q_temp=(1.0, 2.5))]), "integer"), (cases.fipuzen([cases.latent(rot=5)]), "rotated"),
               (cases.fipuzen([cases.latent(kv_rank=5000)]), "latent"), (cases.fipuzen([cases.lightning(heads=3, decay=(0.5,))]), "decay"),
               (cases.fipuzen([(cases.latent(), cases.moe(top=9, experts=4, identity=2))]), "experts"),
               (cases.fipuzen([(cases.latent(), {"kind": "dense", "ff": 8})]), "feed-forward"),
               (cases.fipuzen([{"type": "retention", "mixer": {}}]), "unknown mixer"),
               (cases.fipuzen([(cases.latent(), {**cases.moe(), "expert": {}})]), "ff"),
               (cases.pudadra([(cases.differential(heads=5, kv_heads=2), None)]), "multiple"),
               (cases.pudadra([(cases.differential(window=0), None)]), "mask"), (cases.pudadra([(cases.windowed_latent(window=0), None)]), "mask"),
               (cases.pudadra([(cases.differential(window=2.5), None)]), "integer"), (cases.pudadra([(cases.differential(conv=65), None)]), "taps"),
               (cases.pudadra([(cases.differential(rot=26), None)]), "rotated"), (cases.pudadra([(cases.differential(softcap=-1.0), None)]), "bound"),
               (cases.pudadra([(cases.differential(scaling={"factor": 2.0, "low": 3.0, "high": 3.0, "original": 9}), None)]), "scaling"),
               (cases.pudadra([(cases.differential(), cases.grouped_moe(8, 3, 1, 1))]), "groups"),
               (cases.pudadra([(cases.differential(), cases.grouped_moe(8, 4, 1, 3))]), "groups"),
               (cases.pudadra([(cases.differential(), {"kind": "nosuch"})]), "feed-forward"),
               ({k: v for k, v in cases.CONFIGS["two maps"].items() if k != "residual_mult"}, "residual_mult"),
               (cases.desalix([(cases.chunked(heads=5, kv_heads=2), None)]), "multiple"), (cases.desalix([(cases.chunked(chunk=-3), None)]), "mask"),
               (cases.desalix([(cases.chunked(chunk=2.5), None)]), "integer"), (cases.desalix([(cases.chunked(vdim=9), None)]), "rotated"),
               (cases.desalix([(cases.chunked(rot=26), None)]), "rotated"), (cases.desalix([(cases.chunked(), cases.gated_moe(4, 5))]), "uses"),
               (cases.desalix([(cases.chunked(), cases.gated_moe(limit=-1.0))]), "limit"), (cases.desalix([(cases.chunked(), cases.dense())]), "feed-forward"),
               (cases.desalix([(cases.latent(), None)]), "unknown mixer"),
               *((cases.desalix([(cases.chunked(), None)] * 2, loop=l), "loop") for l in ((0, 3, 2), (1, 1, 2), (-1, 1, 2), (0, 1, 0))),
               ({k: v for k, v in cases.CONFIGS["chunks"].items() if k != "embedding"}, "embedding")]
        for cfg, word in bad:
            with pytest.raises(P.NanoflowPipelineError, match=word):
                _set(tmp_path, cfg)
        with pytest.raises(P.NanoflowPipelineError, match="dtype"):
            _set(tmp_path, good, dtype="float16")
    finally:
        P.setModelConfig(_llama_config(tmp_path))       # the process's other tests configure Llama models
    assert P.stackStateSlots() == 0


def _llama_config(tmp_path):
    import os
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    return os.path.join(root, "nanoflow_amd", "config_all", "llama3-8B.json")


def test_pipeline_file_names_a_stack_model(tmp_path):
    cfg = cases.CONFIGS["odd"]
    stack_models.save_model(str(tmp_path / "m"), cfg, {"head": np.zeros((2, 2), np.float32)})
    base = {"model_configs": {"max_batch_size": 32, "kv_pages": 12, "state_slots": 5, "dtype": "float32"}, "pipeline_configs": {}}
    try:
        for model in (cfg, {"path": "m"}, {"path": str(tmp_path / "m")}):
            f = tmp_path / "pipeline.json"
            f.write_text(json.dumps({"model": model, **base}))
            P.setModelConfig(str(f))
            assert P.stackStateSlots() == 5 and P.maxPageNum() == 12
    finally:
        P.setModelConfig(_llama_config(tmp_path))


@pytest.mark.parametrize("name,some", [("mixed", ("embed", "l1.mix.left.sink", "l1.mix.right.u")),
                                       ("chunks", ("loop.step", "l0.norm1b", "final.norm", "l3.mlp.shared.gate")), ("two maps", ("embed", "l0.mix.q.conv", "l4.mix.lq2", "l1.mlp.shared.sg")), ("five layers", ("side.embed", "l0.mix.q.b", "l2.mlp.e1.down", "l2.mlp.correction"))])
def test_safetensors_of_random_tensors_reads_back(tmp_path, name, some):
    from safetensors import safe_open
    cfg = cases.CONFIGS[name]
    bits, _ = cases.tensors(cfg)
    stack_models.save_model(str(tmp_path), cfg, bits)
    with safe_open(str(tmp_path / "model.safetensors"), "pt") as f:
        assert set(f.keys()) == set(bits) == set(stack_models.tensor_shapes(cfg))
        for k in some:
            np.testing.assert_array_equal(f.get_tensor(k).float().numpy(), stack_models.bits_to_f32(bits[k]))


def _drive(former, cycles=400):
    """Runs the scheduler without a GPU; yields the formed batches."""
    for _ in range(cycles):
        st = former.state()
        if st["queued"] + st["decoding"] + st["prefilling"] == 0:
            return
        former.schedule()
        b = former.form()
        yield b, former.state_slots()
        former.advance(0.0)


def test_state_slots_limit_admission_and_are_used_again():
    f = P.BatchFormer(64, 16, 40, 40, 40, 0, 20, 6)
    f.set_state_slots(3)
    rng = np.random.default_rng(0)
    for i in range(11):
        f.add_request(i, rng.integers(0, 9, int(rng.integers(1, 70))), int(rng.integers(2, 9)))
    seen, most = set(), 0
    for b, slots in _drive(f):
        n = b["decodePrefillBorder"] + b["prefillNum"]
        assert len(slots) == n and len(set(slots.tolist())) == n and set(slots.tolist()) <= {0, 1, 2}
        seen |= set(slots.tolist())
        most = max(most, n)
    assert f.state()["retired"] == 11 and most == 3 and seen == {0, 1, 2}
    f.close()


def test_a_request_keeps_its_slot_and_pages_until_it_retires():
    f = P.BatchFormer(64, 16, 24, 24, 24, 0, 30, 8)
    f.set_state_slots(4)
    for i, n in enumerate((50, 20, 33)):
        f.add_request(i, np.zeros(n, np.int32), 5 + i)
    owner = {}
    for b, slots in _drive(f):
        for r, s in enumerate(slots.tolist()):
            first_page = int(b["kv_indices"][b["kv_indptr"][r]])
            start = b["per_token_offset"][b["input_indptr"][r]] == 0
            assert start or owner[s] == first_page          # the request in a slot is recognised by its first page
            owner[s] = first_page
    f.close()


def test_without_slots_nothing_changes():
    f = P.BatchFormer(64, 16, 40, 40, 40, 0, 20, 6)
    f.add_request(0, np.zeros(10, np.int32), 3)
    for b, slots in _drive(f):
        assert len(slots) == 0
    f.close()


def test_every_entry_point_has_declared_argument_types():
    """Without them ctypes hands pointers over as 32-bit integers."""
    from nanoflow_amd import kernels as K
    without = {name for name in K.SYMBOLS if getattr(K.lib(), name).argtypes is None}
    assert without <= {"nf_abi_version", "nf_last_error"}, without      # these take none


def test_argument_errors_without_a_gpu():
    from nanoflow_amd import kernels as K
    l = K.lib()
    a = K.RecurrenceArgs(dtype=K.BF16, kind=7, heads=1, dim=8, vdim=8)
    assert l.nf_linear_recurrence(ctypes.byref(a), None) == -1 and b"kind" in l.nf_last_error()
    w = K.WindowAttentionArgs(kv=K.KVLayout(K.BF16, 4, 3, 8, 8, 32, 16, 16, 1))
    assert l.nf_window_attention(ctypes.byref(w), None) == -1 and b"kv heads" in l.nf_last_error()
    assert l.nf_gemm_nk_bf16(None, None, None, 4, 12, 64, None, 0, None) == -1
    r = K.ResidualArgs(rows=4, width=8, ld=8, y_dtype=K.F32, shares=17)
    assert l.nf_residual_rows(ctypes.byref(r), None) == -1 and b"17 shares" in l.nf_last_error()
    r = K.ResidualArgs(rows=4, width=8, ld=8, y_dtype=K.F32, shares=1, next=K.Norm(kind=9))
    assert l.nf_residual_rows(ctypes.byref(r), None) == -1 and b"norm 9" in l.nf_last_error()
    w.kv = K.KVLayout(K.BF16, 4, 2, 8, 8, 32, 16, 16, 3)
    assert l.nf_window_attention(ctypes.byref(w), None) == -1 and b"3 maps" in l.nf_last_error()
    conv = K.ShortConv(taps=65)
    assert l.nf_conv_state(K.BF16, None, 8, ctypes.byref(conv), None, 0, 1, None) == -1 and b"taps" in l.nf_last_error()
    route = lambda **kw: l.nf_route(ctypes.byref(K.RouteArgs(**{**dict(shares=1, ld=16, rows=4, outputs=8, experts=6, top=2, scale=1.0), **kw})),
                                    ctypes.byref(K.Routing(tile_rows=64)), None)
    assert route(top=9) == -1 and b"top 9" in l.nf_last_error()                                   # of 8 outputs
    assert route(groups=3, keep_groups=1) == -1 and b"groups" in l.nf_last_error()                # that do not divide them
    assert route(groups=4, keep_groups=1, top=3) == -1 and b"top 3" in l.nf_last_error()          # of a group of two
    assert route(ld=8, always=1) == -1 and b"ld=8" in l.nf_last_error()                           # no room for its gate
    g = K.GroupedGemmArgs(dtype=K.BF16, act=K.ACT_SILU, groups=2, M=4, N=8, K=8, lda=8, ldd=8)
    assert l.nf_gemm_grouped(ctypes.byref(g), None) == -1 and b"activation" in l.nf_last_error()
    g = K.GroupedGemmArgs(dtype=K.BF16, groups=2, M=4, N=8, K=8, lda=8, ldd=4)
    assert l.nf_gemm_grouped(ctypes.byref(g), None) == -1 and b"strides" in l.nf_last_error()
    g = K.GroupedGemmArgs(dtype=K.BF16, groups=2, M=4, N=8, K=8, lda=8, ldd=8, weigh=1)
    assert l.nf_gemm_grouped(ctypes.byref(g), None) == -1 and b"weights" in l.nf_last_error()
    w = K.WindowAttentionArgs(kv=K.KVLayout(K.BF16, 4, 2, 8, 8, 32, 16, 16, 1), out_ld=32, out_rot=K.Rotation(None, 8, 0))
    assert l.nf_window_attention(ctypes.byref(w), None) == -1 and b"turned back" in l.nf_last_error()
    assert route(scores=2) == -1 and b"scores" in l.nf_last_error()
    lay = K.LatentLayout()
    assert l.nf_latent_layout_of(K.BF16, 4, 20, 6, 16, ctypes.byref(lay)) == 0 and (lay.rank_pad, lay.row_ld) == (24, 64)
    assert l.nf_latent_layout_of(K.BF16, 4, 4000, 6, 16, ctypes.byref(lay)) == -1
    lay.row_ld = 8
    a = K.LatentAttentionArgs(layout=lay)
    assert l.nf_latent_attention(ctypes.byref(a), None) == -1
    assert l.nf_recurrence_state_elements(20, 40) == 32 * 48
