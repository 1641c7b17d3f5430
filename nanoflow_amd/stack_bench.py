"""Prefill and decode throughput of layer-stack models (random weights) at sizes that resemble real
models' layers, beside the Llama-type pipeline at the same width, feed-forward, depth and vocabulary (of a mixture:
the feed-forward a token uses on average).

All sides run the same batches: a prefill iteration of 2048 tokens (two prompts of 1024), one of a single 2048-token
prompt, and decode iterations of 16, 64 and 256 requests at a context of 1024 whose caches and states were filled by prefilling
them.  An iteration is one run(): embedding ... sampler, replayed from a hipGraph; update data is staged before."""
from __future__ import annotations

import time

import numpy as np

VOCAB = 32768


def stack_config(width, ff, pairs=2, heads=None):
    """`pairs` x (a retention layer, a parallel layer); heads of 128 (attention 4 query heads per kv head), recurrence
    heads of 64."""
    n = width // 128
    retention = {"heads": n, "dim": 128, "vdim": 128, "decay": [1.0 - 2.0 ** (-5 - 3.0 * h / n) for h in range(n)],
                 "rot": {"dims": 128, "base": 1e4}}
    parallel = {"left": {"heads": n, "kv_heads": n // 4, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                         "mask": {"size": 512, "keep_first": 16}, "rot": {"dims": 128, "base": 1e4}},
                "right": {"heads": width // 64, "dim": 64}, "left_scale": 1.0, "right_scale": 0.5}
    mlp = {"kind": "dense", "ff": ff}
    layers = []
    for _ in range(pairs):
        layers += [{"type": "retention", "mixer": retention, "mlp": mlp}, {"type": "parallel", "mixer": parallel, "mlp": mlp}]
    return {"architecture": "Zovovik", "width": width, "vocab": VOCAB, "max_positions": 4096, "norm": {"eps": 1e-5}, "layers": layers}


def fipuzen_config(width, ff):
    """(attention, latent attention, lightning, attention), heads of 128 (4 query heads per kv head, latents of 512 + 64 rotated),
    each with 32 experts of a quarter of `ff` and 8 identity experts of which a token uses 5."""
    n = width // 128
    attention = {"heads": n, "kv_heads": n // 4, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "q_temp": {"coef": 0.1, "every": 512}}
    latent = {"heads": n, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "scale": 192 ** -0.5, "rot": {"dims": 64, "base": 1e4}}
    lightning = {"heads": n, "dim": 128, "vdim": 128, "decay": [1.0 - 2.0 ** (-5 - 3.0 * h / n) for h in range(n)]}
    moe = {"kind": "moe", "expert": {"ff": ff // 4}, "router": {"experts": 32, "identity": 8, "top": 5, "scale": 2.0}}
    layers = [{"type": t, "mixer": m, "mlp": moe} for t, m in
              (("attention", attention), ("latent_attention", latent), ("lightning", lightning), ("attention", attention))]
    return {"architecture": "Fipuzen", "width": width, "vocab": VOCAB, "token_side": {"dim": 256}, "norm": {"eps": 1e-5}, "layers": layers}


def pudadra_config(width, ff):
    """(attention, attention, latent attention, attention), all over the last 512 tokens: two maps of 64 over values of 128 (4 query
    heads per kv head, convolutions of 4 taps), latents of 512 + 64 rotated; first a dense feed-forward of `ff`, then 32 experts
    of a quarter of it in 8 groups, of which a token uses 4 out of 4 groups, and a shared one."""
    n, window = width // 128, {"size": 512}
    attention = {"heads": n, "kv_heads": n // 4, "dim": 64, "vdim": 128, "scale": 64 ** -0.5, "softcap": 30.0, "conv": 4, "diff": 0.4, "mask": window,
                 "rot": {"dims": 64, "base": 5e5, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
    latent = {"heads": n, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "scale": 192 ** -0.5, "mask": window, "rot": {"dims": 64, "base": 1e4}}
    moe = {"kind": "moe", "expert": {"ff": ff // 4}, "shared": {"ff": ff // 4},
           "router": {"experts": 32, "groups": {"count": 8, "keep": 4}, "top": 4}}
    layers = [("attention", attention, {"kind": "dense", "ff": ff}), ("attention", attention, moe), ("latent_attention", latent, moe),
              ("attention", attention, moe)]
    return {"architecture": "Pudadra", "width": width, "vocab": VOCAB, "residual_mult": 0.5, "logit_scale": 0.5, "norm": {"eps": 1e-5},
            "layers": [{"type": t, "mixer": m, "mlp": f} for t, m, f in layers]}


def desalix_config(width, ff):
    """Three layers of attention in chunks of 1536 (heads of 128, 4 query heads per kv head), the middle one passed twice; 32 experts
    of a quarter of `ff`, 4 of them per token, and a shared one."""
    n, expert = width // 128, {"ff": ff // 4, "limit": 7.0}
    attention = {"heads": n, "kv_heads": n // 4, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "mask": {"size": 1536}, "rot": {"dims": 64, "base": 5e5}}
    moe = {"kind": "moe", "expert": expert, "shared": expert, "router": {"experts": 32, "top": 4}}
    return {"architecture": "Desalix", "width": width, "vocab": VOCAB, "embedding": {"scale": 8.0}, "norm": {"eps": 1e-5},
            "loop": {"start": 1, "stop": 2, "times": 2}, "layers": [{"type": "attention", "mixer": attention, "mlp": moe}] * 3}


# side -> configuration of a layer-stack model; "llama" is the other kind
DESIGNS = {"stack": stack_config, "fipuzen": fipuzen_config, "pudadra": pudadra_config, "desalix": desalix_config}
SIZES = {"2048": (2048, 8192), "4096": (4096, 14336)}


def _sub_prefill(b, first, count, length, vocab, seed):
    """The batch that prefills `length` tokens of requests [first, first + count) of batch b into their own pages."""
    from nanoflow_amd import synth
    s = synth.make_batch([], [(0, length)] * count, vocab, seed=seed)
    n_pages = (length + 15) // 16
    s.kv_indices = np.concatenate([b.kv_indices[b.kv_indptr[r]:b.kv_indptr[r] + n_pages] for r in range(first, first + count)]).astype(np.int32)
    return s


def _time(run, steps, warmup):
    """Milliseconds per iteration: `steps` of them in up to five blocks, the median block (the runtime pauses once in a while for
    tens of milliseconds, which is not the model's)."""
    import torch
    for _ in range(warmup):
        run()
    per_block, times = max(steps // 5, 1), []
    for first in range(0, steps, per_block):
        n = min(per_block, steps - first)
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        for _ in range(n):
            run()
        torch.cuda.synchronize()
        times.append((time.perf_counter() - t0) / n * 1e3)
    return float(np.median(times))


def _cases():
    from nanoflow_amd import synth
    return {"prefill 2 x 1024": synth.make_batch([], [(0, 1024)] * 2, VOCAB, seed=1),
            "prefill 1 x 2048": synth.make_batch([], [(0, 2048)], VOCAB, seed=2),
            **{f"decode {n} at 1024": synth.make_batch([1024] * n, [], VOCAB, seed=3 + n) for n in (16, 64, 256)}}


def run_sizes(steps=20, warmup=4, sizes=tuple(SIZES), cases=None, sides=("stack", "llama"), graph=True):
    """One record per size: milliseconds and tokens/s of every case on every side."""
    from nanoflow_amd import engine, synth, pllm_python as P
    out = []
    for size in sizes:
        width, ff = SIZES[size]
        layers = 4
        batches = {k: b for k, b in _cases().items() if cases is None or k in cases}
        pages = max(b.num_pages for b in _cases().values())
        rec = {"width": width, "ff": ff, "layers": layers, "cases": {}}
        for side in sides:
            if side in DESIGNS:
                cfg = DESIGNS[side](width, ff)
                loop = cfg.get("loop") or {"start": 0, "stop": 0, "times": 1}
                assert len(cfg["layers"]) + (loop["times"] - 1) * (loop["stop"] - loop["start"]) == layers
                e = engine.StackEngine(cfg, global_batch=2048, kv_pages=pages, state_slots=256, rank=64)
            else:
                shape = synth.ModelShape(hidden=width, Hq=width // 128, Hkv=width // 512, d=128, ffn=ff, vocab=VOCAB, layers=layers)
                e = engine.Engine(shape, P.PipelineType.NON_OVERLAP_LOCAL, global_batch=2048, nano1=1024, kv_pages=pages, weight_layout="col")
            P.setGraphMode(graph)

            def stage(b, slots):
                if side in DESIGNS:
                    e.update(b, slots, decode_tokens=b.input_tokens[:b.decodePrefillBorder] if b.decodePrefillBorder else None)
                else:
                    e.update(b, keep_token_list=np.ones(b.decodePrefillBorder, np.int32))

            for name, b in batches.items():
                n = b.decodePrefillBorder
                for first in range(0, n, 2):      # histories of the decode requests
                    stage(_sub_prefill(b, first, 2, 1024, VOCAB, 7 + first), np.arange(first, first + 2))
                    e.run()
                if side == "llama" and n:
                    # its decode rows continue the last iteration's requests: one that has all n of them
                    one = synth.make_batch([], [(0, 1)] * n, VOCAB, seed=9)
                    one.kv_indices = b.kv_indices[b.kv_indptr[:-1]].astype(np.int32)
                    e.update(one)
                    e.run()
                stage(b, np.arange(b.req_num))
                ms = _time(e.run, steps, warmup)
                rec["cases"].setdefault(name, {})[side] = {"ms": round(ms, 4), "tokens_per_s": round(b.tokens / ms * 1e3)}
            P.setGraphMode(False)
            e.close()
        out.append(rec)
    return out


if __name__ == "__main__":
    import argparse
    import json
    ap = argparse.ArgumentParser(description=__doc__)
    ap.add_argument("--size", choices=list(SIZES), action="append")
    ap.add_argument("--case", action="append")
    ap.add_argument("--side", choices=[*DESIGNS, "llama"], action="append")
    ap.add_argument("--steps", type=int, default=20)
    ap.add_argument("--eager", action="store_true")
    a = ap.parse_args()
    for r in run_sizes(a.steps, 4, a.size or tuple(SIZES), a.case, a.side or ("stack", "llama"), not a.eager):
        print(json.dumps(r))
