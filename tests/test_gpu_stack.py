"""Layer-stack models through the framework: StackEngine, replay, the batch former and the serving loop, against the plain
implementation."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")
pytestmark = pytest.mark.gpu

from nanoflow_amd import engine, pllm_python as P, stack_models  # noqa: E402
from oracle import stack_oracle as S  # noqa: E402

import stack_cases as cases  # noqa: E402

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# rms error of a row of logits over the rms of all logits.  bf16 rows are 0.3-0.8 % off at the median; one whose head
# outputs nearly cancel before their norm (a first token that does not answer its own key) is off by several.
TOL = {"float32": 4e-5, "bfloat16": 0.12}
# Where a router chooses, rounding to bf16 now and then lets another expert in: single rows are off by what one small
# expert gives, and the rows as a whole are as close as elsewhere.
TOL_CHOICE = 0.5


@pytest.fixture(scope="module", autouse=True)
def _gpu():
    assert torch.cuda.is_available()
    P.lib()
    yield
    P.setModelConfig(os.path.join(ROOT, "nanoflow_amd", "config_all", "llama3-8B.json"))   # later tests configure Llama models


_models = {}


def model(name, seed=0):
    """(configuration, bit patterns, floats) of a small model whose layers count."""
    if (name, seed) not in _models:
        cfg = cases.CONFIGS[name]
        bits, t = cases.tensors(cfg, seed)
        _models[name, seed] = (cfg, bits, t)
    return _models[name, seed]


def make(name, dtype, batch=256, pages=80, slots=6, **kw):
    cfg, bits, _ = model(name)
    return engine.StackEngine(cfg, dtype=dtype, global_batch=batch, kv_pages=pages, state_slots=slots, weights=bits, **kw)


def sequences(name, lengths, seed=0):
    cfg, _, t = model(name)
    rng = np.random.default_rng(seed)
    toks = [rng.integers(0, cfg["vocab"], n) for n in lengths]
    return toks, [S.forward(cfg, t, x) for x in toks]


def check(got, want, dtype, what="", choice=False):
    scale = np.sqrt((want ** 2).mean())
    d = got - want
    err = np.sqrt((d ** 2).mean(axis=-1)) / scale
    tol = TOL_CHOICE if choice and dtype == "bfloat16" else TOL[dtype]
    assert np.isfinite(got).all() and err.max() <= tol, f"{what}: {err.max():.2e} at {int(err.argmax())}"
    if dtype == "bfloat16" and len(err) >= 16:
        assert np.median(err) <= 0.02, f"{what}: median {np.median(err):.2e}"


def chooses(name):
    return any((l.get("mlp") or {}).get("kind") == "moe" for l in cases.CONFIGS[name]["layers"])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(cases.CONFIGS))
def test_whole_prompts_and_every_layer(name, dtype):
    cfg, _, t = model(name)
    (tok,), _ = sequences(name, [130])
    want, layers = S.forward(cfg, t, tok, want_layers=True)
    with make(name, dtype, keep_layers=True) as e:
        r = e.replay()
        got = r.step([("a", tok, range(len(tok)))], e.vocab)["a"]
        for i in range(len(layers)):
            check(P.stackLayerOutput(i), layers[i], dtype, f"layer {i}", chooses(name))
        check(got, want, dtype, "logits", chooses(name))
        r.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "odd", "wide heads", "five layers", "odd sizes", "large heads", "one expert", "two maps", "odd maps", "large maps",
                                  "window of one map", "chunks", "odd chunks", "large chunks", "chunk of one", "one chunk"])
def test_token_by_token_and_portions_agree_with_the_whole(name, dtype):
    (tok,), (want,) = sequences(name, [90])
    with make(name, dtype) as e:
        r = e.replay()
        for sizes in ([1] * 90, [2] * 45, [3, 2, 16, 29, 1, 2, 37], [15, 1, 17, 31, 26], [64, 2, 2, 2, 20], [89, 1]):
            at = 0
            for n in sizes:
                got = r.step([("a", tok[at:at + n], range(n))], e.vocab)["a"]
                check(got, want[at:at + n], dtype, f"{sizes} at {at}", chooses(name))
                at += n
            assert at == 90
            r.end("a")
            assert r.state() == {"live": 0, "free_pages": 80, "free_slots": 6}
        r.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "five layers", "two maps", "chunks"])
def test_unequal_requests_beside_each_other_and_slots_used_again(name, dtype):
    """Portions beside single tokens, requests that pause, end and leave their pages and slots to others."""
    lengths = [140, 1, 33, 75, 64, 2, 110, 17, 48, 90]
    toks, wants = sequences(name, lengths, seed=4)
    rng = np.random.default_rng(11)
    with make(name, dtype, pages=24, slots=3) as e:
        r = e.replay(24, 3)
        waiting, live, at, steps, mixed = list(range(len(toks))), [], {}, 0, 0
        while waiting or live:
            while waiting and len(live) < 3 and sum((lengths[i] + 15) // 16 for i in live + [waiting[0]]) <= 24:
                at[waiting[0]] = 0
                live.append(waiting.pop(0))
            entries = []
            for i in live:
                if len(live) > 1 and rng.random() < 0.2 and not (i == live[-1] and not entries):
                    continue                              # left out of this step
                n = 1 if at[i] and rng.random() < 0.4 else int(rng.integers(1, 40))
                n = min(n, lengths[i] - at[i])
                entries.append((i, toks[i][at[i]:at[i] + n], range(n)))
            rng.shuffle(entries)
            mixed += len({len(t) == 1 for _, t, _ in entries}) == 2
            res = r.step(entries, e.vocab)
            for i, t, _ in entries:
                check(res[i], wants[i][at[i]:at[i] + len(t)], dtype, f"request {i} at {at[i]}", chooses(name))
                at[i] += len(t)
                if at[i] == lengths[i]:
                    r.end(i)
                    live.remove(i)
            steps += 1
            assert steps < 200
        assert mixed > 3 and r.state() == {"live": 0, "free_pages": 24, "free_slots": 3}
        r.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "five layers", "two maps", "chunks"])
def test_long_decoding(name, dtype):
    (tok,), (want,) = sequences(name, [330], seed=8)
    with make(name, dtype) as e:
        r = e.replay()
        check(r.step([("a", tok[:40], [0, 39])], e.vocab)["a"], want[[0, 39]], dtype)
        rows = []
        for i in range(40, 330):
            rows.append(r.step([("a", tok[i:i + 1], [0])], e.vocab)["a"])
            check(rows[-1], want[i:i + 1], dtype, f"position {i}", chooses(name))
        check(np.concatenate(rows), want[40:], dtype, "all", chooses(name))
        r.close()


@pytest.mark.parametrize("name", ["mixed", "five layers", "two maps", "chunks"])
def test_many_rows_and_only_some_logits(name):
    """A step of more rows than the small-batch paths take, logits of a few places only."""
    (tok,), (want,) = sequences(name, [580], seed=9)
    for dtype in TOL:
        with make(name, dtype, batch=1200, pages=90) as e:
            r = e.replay()
            some = [0, *range(100, 140), 579]
            res = r.step([("a", tok, some), ("b", tok[:570], []), ("c", tok[:1], [0])], e.vocab)
            check(res["a"], want[some], dtype, "a", chooses(name))
            check(res["c"], want[:1], dtype, "c", chooses(name))
            check(r.step([("b", tok[570:571], [0])], e.vocab)["b"], want[570:571], dtype, "b", chooses(name))
            r.close()


def test_replay_errors_are_reported():
    with make("mixed", "bfloat16", pages=6, slots=2) as e:
        r = e.replay(6, 2)
        with pytest.raises(P.NanoflowPipelineError, match="vocabulary"):
            r.step([("a", [e.vocab], [])], e.vocab)
        r.close()
        r = e.replay(6, 2)
        with pytest.raises(P.NanoflowPipelineError, match="memory"):
            r.step([("a", np.zeros(100, int), [])], e.vocab)
        r.close()
        r = e.replay(6, 2)
        with pytest.raises(P.NanoflowPipelineError, match="slot"):
            r.step([(i, [1], []) for i in range(3)], e.vocab)
        r.close()
    with pytest.raises(P.NanoflowPipelineError, match="missing"):
        cfg, bits, _ = model("mixed")
        engine.StackEngine(cfg, global_batch=8, kv_pages=4, state_slots=1, weights={k: v for k, v in bits.items() if k != "l1.norm1"})
    with pytest.raises(P.NanoflowPipelineError, match="shape"):
        engine.StackEngine(cfg, global_batch=8, kv_pages=4, state_slots=1, weights={**bits, "head": bits["head"][:-1]})


def greedy(cfg, t, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(S.forward(cfg, t, seq)[-1].argmax()))
    return seq[len(prompt):]


@pytest.mark.parametrize("name", ["odd", "odd sizes", "five layers", "odd maps", "two maps", "odd chunks", "chunks"])
def test_greedy_generation_through_the_scheduler(name):
    """The batch former and the serving loop (fp32: the sampled ids are the plain implementation's), eagerly and replayed from
    graphs; more requests than slots."""
    cfg, bits, t = model(name)
    rng = np.random.default_rng(2)
    reqs = [(rng.integers(0, cfg["vocab"], n), out) for n, out in ((30, 8), (5, 10), (61, 6), (1, 9), (17, 7))]
    want = [greedy(cfg, t, p, n) for p, n in reqs]
    for graphs in (False, True):
        with make(name, "float32", batch=40, pages=24, slots=3) as e:
            P.setGraphMode(graphs)
            f = e.former(30, 8)
            for i, (p, n) in enumerate(reqs):
                f.add_request(i, p, n)
            f.serve(0, 200)
            P.setGraphMode(False)
            assert f.state()["retired"] == len(reqs)
            for k in range(len(reqs)):
                i, out = f.retired_output(k)
                out = [int(x) for x in out if x >= 0]
                # retirement is by length and one iteration late: the sample of a request's last iteration replaces
                # the one before it, as in the other models' loop
                n = reqs[i][1]
                assert len(out) == n - 1 and out[:-1] == want[i][:n - 2] and out[-1] in want[i][n - 2:n], (i, out, want[i])
            f.close()


@pytest.mark.parametrize("name", ["mixed", "five layers", "two maps", "chunks"])
def test_graph_replays_equal_eager_iterations(name):
    from nanoflow_amd import synth
    cfg, bits, _ = model(name)
    b = synth.make_batch([20, 50, 3], [(0, 70), (30, 40)], cfg["vocab"], seed=3)
    h, reqs = cases.history_batch(b)
    slots = np.array([3, 0, 4, 1, 2], np.int32)
    logits = []
    for graphs in (False, True):
        with make(name, "bfloat16") as e:
            P.setGraphMode(graphs)
            runs = []
            for _ in range(4):                       # eager, captured, replayed, replayed
                h.input_tokens = np.arange(h.tokens, dtype=np.int32) % cfg["vocab"]
                e.update(h, slots[reqs])
                e.run()
                e.update(b, slots, decode_tokens=b.input_tokens[:3])
                e.run()
                runs.append(P.getLogits())
            if graphs:
                assert P.getGraphCounters()["replayed"] >= 2
            P.setGraphMode(False)
            logits.append(runs)
    for run in logits[0][1:] + logits[1]:
        np.testing.assert_array_equal(run, logits[0][0])


@pytest.mark.parametrize("name", ["mixed", "odd sizes", "two maps", "chunks"])
def test_trace_program(name, tmp_path):
    """bin/trace_run on a model directory: steps on standard input, logits in files."""
    cfg, bits, _ = model(name)
    stack_models.save_model(str(tmp_path / "m"), cfg, bits)
    toks, wants = sequences(name, [50, 20], seed=6)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[0][:30].tolist(), "want": [0, 29]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": toks[1].tolist(), "want": []}, {"id": "a", "tokens": [int(toks[0][30])], "want": [0]}],
              "end": ["b"]},
             {"step": 2, "entries": [{"id": "b", "tokens": toks[1].tolist(), "want": [19]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": toks[0][31:].tolist(), "want": [18]}], "end": ["a"]}]
    want = {0: wants[0][[0, 29]], 1: wants[0][[30]], 2: wants[1][[19]], 3: wants[0][[49]]}
    for dtype in TOL:
        out = tmp_path / dtype
        out.mkdir()
        p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", dtype, "--out", str(out),
                            "--max-tokens", "128"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
        assert p.returncode == 0, p.stderr[-2000:]
        assert [l for l in p.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
        for i, w in want.items():
            check(np.fromfile(out / f"{i}.f32", "<f4").reshape(w.shape), w, dtype, f"step {i}", chooses(name))


@pytest.mark.parametrize("name", ["odd", "odd sizes", "odd maps", "odd chunks"])
def test_serve_command_line(name, tmp_path):
    cfg, bits, t = model(name)
    stack_models.save_model(str(tmp_path / "m"), cfg, bits)
    (tmp_path / "pipeline.json").write_text(json.dumps({
        "model": {"path": "m"}, "model_configs": {"dtype": "float32", "kv_pages": 32, "state_slots": 4, "max_batch_size": 64},
        "pipeline_configs": {"global_batch_size": 64}, "serve_configs": {"pipeline_type": "LAYER_STACK"}}))
    (tmp_path / "trace.csv").write_text("idx,input_len,output_len,arrival\n" + "".join(f"{i},{n},6,0\n" for i, n in enumerate((12, 40, 3))))
    p = subprocess.run([sys.executable, "-m", "nanoflow_amd.serve", "-t", str(tmp_path / "trace.csv"), "-c", str(tmp_path / "pipeline.json"),
                        "-r", "60", "-s", "0", "-o", str(tmp_path / "out")], cwd=ROOT, capture_output=True, text=True, timeout=110)
    assert p.returncode == 0, p.stderr[-2000:]
    lines = [json.loads(l) for l in (tmp_path / "out.req_tokens").read_text().splitlines()]
    assert len(lines) == 3
    for n, l in zip((12, 40, 3), lines):
        assert l[:n] == list(range(n)) and len(l) > n + 2
        assert l[n:-1] == greedy(cfg, t, range(n), len(l) - n - 1)      # (the last one: see the scheduler's test)
