"""Shared by the tests of layer-stack models: small configurations, batches over permuted pages."""
import numpy as np

from nanoflow_amd import stack_models, synth


def retention(heads=3, dim=24, vdim=40, rot=16, base=500.0, decay=(0.5, 0.97, 1.0)):
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)[:heads],
                                           "rot": {"dims": rot, "base": base}}}


def parallel(heads=6, kv_heads=2, dim=32, vdim=48, window=21, keep=5, scale=0.2, rot=20, base=300.0, right_heads=3,
             right_dim=20, left_scale=0.7, right_scale=1.6):
    return {"type": "parallel", "mixer": {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                 "mask": {"size": window, "keep_first": keep}, "rot": {"dims": rot, "base": base}},
        "left_scale": left_scale, "right": {"heads": right_heads, "dim": right_dim}, "right_scale": right_scale}}


def config(layers, width=104, vocab=211, ff=88, eps=1e-5, max_positions=600):
    """layers: mixers, each with its feed-forward width (None: no feed-forward) or the default one."""
    out = []
    for entry in layers:
        mixer, f = entry if isinstance(entry, tuple) else (entry, ff)
        out.append({**mixer, "mlp": None if f is None else {"kind": "dense", "ff": f}})
    return {"architecture": "Zovovik", "width": width, "vocab": vocab, "max_positions": max_positions, "norm": {"eps": eps}, "layers": out}


def attention(heads=6, kv_heads=2, dim=24, vdim=40, scale=0.25, q_temp=(0.7, 16)):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                                           "q_temp": q_temp and {"coef": q_temp[0], "every": q_temp[1]}}}


def latent(heads=5, dim=24, rot=12, vdim=20, kv_rank=36, scale=0.2, base=700.0):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": kv_rank,
                                                  "scale": scale, "rot": {"base": base, "dims": rot}}}


def lightning(heads=3, dim=16, vdim=24, decay=(0.6, 0.97, 0.999)):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)[:heads]}}


def moe(experts=5, identity=2, top=3, ff=40, scale=1.5):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "identity": identity, "top": top, "scale": scale}}


def fipuzen(layers, width=104, vocab=211, side=20, eps=1e-5, mlp=None):
    """layers: mixers, each alone or with its feed-forward (None: none)."""
    out = []
    for entry in layers:
        mixer, f = entry if isinstance(entry, tuple) else (entry, mlp or moe())
        out.append({**mixer, "mlp": f})
    return {"architecture": "Fipuzen", "width": width, "vocab": vocab, "token_side": {"dim": side}, "norm": {"eps": eps}, "layers": out}


SCALING = {"factor": 6.0, "low": 1.0, "high": 3.0, "original": 300}


def differential(heads=6, kv_heads=2, dim=24, vdim=40, window=21, rot=16, base=300.0, scaling=SCALING, scale=0.25, softcap=6.0, conv=3, diff=0.4):
    return {"type": "attention", "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": softcap, "conv": conv, "diff": diff,
        "mask": {"size": window}, "rot": {"dims": rot, "base": base, **({"scaling": scaling} if scaling else {})}}}


def windowed_latent(window=37, **kw):
    m = latent(**kw)
    m["mixer"]["mask"] = {"size": window}
    return m


def dense(ff=88):
    return {"kind": "dense", "ff": ff}


def grouped_moe(experts=8, groups=4, keep=2, top=3, ff=40, shared=56):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "groups": {"count": groups, "keep": keep}, "top": top}}
    return {**m, "shared": {"ff": shared}} if shared else m


def pudadra(layers, width=104, vocab=211, eps=1e-5, residual_mult=0.7, logit_scale=0.3):
    """layers: (mixer, feed-forward or None)"""
    return {"architecture": "Pudadra", "width": width, "vocab": vocab, "residual_mult": residual_mult, "logit_scale": logit_scale,
            "norm": {"eps": eps}, "layers": [{**mixer, "mlp": f} for mixer, f in layers]}


def chunked(heads=6, kv_heads=2, dim=24, vdim=40, chunk=21, rot=16, base=300.0, scale=0.3):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                                           "mask": chunk and {"size": chunk}, "rot": {"dims": rot, "base": base}}}


def gated_moe(experts=6, top=2, ff=40, limit=0.6, shared=56, shared_limit=0.9):
    m = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    return {**m, "shared": {"ff": shared, "limit": shared_limit}} if shared else m


def desalix(layers, loop=None, width=104, vocab=211, eps=1e-5, scale=1.7):
    """layers: (mixer, feed-forward or None); loop: (start, stop, times)"""
    return {"architecture": "Desalix", "width": width, "vocab": vocab, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "loop": loop and dict(zip(("start", "stop", "times"), loop)), "layers": [{**mixer, "mlp": f} for mixer, f in layers]}


# sizes that are not multiples of 8, equal and unequal head counts, no feed-forward, a window of one, windows without kept tokens
CONFIGS = {
    "mixed": config([retention(), parallel(), (retention(heads=1, dim=16, vdim=16, rot=16, decay=(0.9,)), None), parallel(
        heads=4, kv_heads=4, dim=16, vdim=16, window=33, keep=0, rot=16, right_heads=1, right_dim=64)]),
    "odd": config([parallel(heads=5, kv_heads=1, dim=18, vdim=10, window=7, keep=3, rot=6, right_heads=2, right_dim=10),
                   retention(heads=2, dim=10, vdim=6, rot=4, decay=(0.8, 0.999))], width=52, vocab=97, ff=70, eps=1e-3),
    "wide heads": config([parallel(heads=2, kv_heads=1, dim=160, vdim=144, window=64, keep=16, rot=64, right_heads=1, right_dim=128),
                          retention(heads=1, dim=96, vdim=128, rot=96, decay=(0.99,))], width=128, ff=160),
    "retention only": config([retention(heads=2, dim=64, vdim=64, rot=32, decay=(0.99, 0.9)), retention(heads=2, dim=32, vdim=96, rot=32)]),
    "five layers": fipuzen([attention(), latent(), lightning(), (latent(heads=2, dim=16, rot=16, vdim=32, kv_rank=64), None),
                            (attention(heads=4, kv_heads=4, dim=32, vdim=16, q_temp=(1.5, 7)), moe(experts=3, identity=0, top=1, scale=1.0))]),
    "odd sizes": fipuzen([latent(heads=3, dim=10, rot=6, vdim=9, kv_rank=21, base=50.0), attention(heads=3, kv_heads=1, dim=18, vdim=10, q_temp=(0.3, 1)),
                          (lightning(heads=2, dim=10, vdim=7, decay=(0.9, 1.0)), moe(experts=7, identity=1, top=5, ff=18))],
                         width=52, vocab=97, side=5, eps=1e-3),
    "large heads": fipuzen([(latent(heads=20, dim=32, rot=32, vdim=48, kv_rank=288), moe(experts=9, identity=3, top=4, ff=72)), lightning(heads=1, dim=96, vdim=128, decay=(0.99,)),
                            attention(heads=2, kv_heads=1, dim=160, vdim=144), (latent(heads=40, dim=16, rot=8, vdim=16, kv_rank=520), None)], width=128),
    "one expert": fipuzen([attention(heads=1, kv_heads=1, dim=8, vdim=8), (lightning(heads=1, dim=16, vdim=16, decay=(0.8,)), moe(1, 0, 1, 8, 1.0)),
                           (latent(heads=1, dim=8, rot=2, vdim=8, kv_rank=8), moe(1, 6, 2, 24))], width=40, side=8),
    "two maps": pudadra([(differential(), dense()), (windowed_latent(), grouped_moe()), (differential(heads=4, kv_heads=4, dim=32, vdim=16, window=70, rot=32,
                                                                                                     conv=4), None),
                         (windowed_latent(heads=2, dim=16, rot=16, vdim=32, kv_rank=64, window=20), dense(70)),
                         (differential(heads=2, kv_heads=1, dim=16, vdim=48, scaling=None, softcap=None, conv=2), grouped_moe(6, 1, 1, 2, 24, None))]),
    "odd maps": pudadra([(windowed_latent(heads=3, dim=10, rot=6, vdim=9, kv_rank=21, base=50.0, window=11), grouped_moe(9, 3, 1, 2, 18, 70)),
                         (differential(heads=3, kv_heads=1, dim=18, vdim=10, window=7, rot=6, conv=5, diff=0.15), grouped_moe(7, 7, 4, 4, 30, 13)),
                         (differential(heads=1, kv_heads=1, dim=7, vdim=5, window=300, rot=2, conv=1, softcap=0.9, scale=1.0), dense(33))],
                        width=51, vocab=97, eps=1e-3, residual_mult=1.0, logit_scale=1.7),
    "large maps": pudadra([(differential(heads=4, kv_heads=2, dim=64, vdim=128, window=60, rot=64, scale=0.125), grouped_moe(16, 4, 3, 5, 72, 72)),
                           (differential(heads=5, kv_heads=1, dim=96, vdim=144, window=33, rot=96, scale=0.1, conv=6), None),
                           (windowed_latent(heads=20, dim=32, rot=32, vdim=48, kv_rank=288, window=50), dense(160)),
                           (differential(heads=2, kv_heads=2, dim=160, vdim=72, window=90, rot=80, scale=0.08), grouped_moe(4, 2, 2, 4, 64, 300))], width=128),
    "window of one map": pudadra([(differential(heads=2, kv_heads=2, dim=8, vdim=8, window=1, rot=8, conv=2), grouped_moe(2, 2, 1, 1, 8, 8)),
                                  (windowed_latent(heads=1, dim=8, rot=2, vdim=8, kv_rank=8, window=1), None),
                                  (differential(heads=9, kv_heads=3, dim=16, vdim=32, window=16, rot=0, conv=9), dense(8))], width=40),
    "chunks": desalix([(chunked(), gated_moe()), (chunked(heads=4, kv_heads=4, dim=32, vdim=16, chunk=50, rot=32), None), (chunked(chunk=16), gated_moe(4, 3, 24)),
                       (chunked(heads=2, kv_heads=1, dim=16, vdim=48, chunk=35, base=90.0), gated_moe(5, 1, 64, 1.5, 20, 0.4))], loop=(1, 3, 3)),
    "odd chunks": desalix([(chunked(heads=5, kv_heads=1, dim=18, vdim=10, chunk=7, rot=6), gated_moe(7, 4, 18, 0.3, 70, 2.0)),
                           (chunked(heads=3, kv_heads=1, dim=9, vdim=6, chunk=40, rot=2, scale=0.8), None),
                           (chunked(heads=2, kv_heads=2, dim=7, vdim=2, chunk=300, rot=0), gated_moe(3, 2, 13, 0.7, None))], loop=(0, 2, 2), width=51, vocab=97,
                          eps=1e-3, scale=0.4),
    "large chunks": desalix([(chunked(heads=4, kv_heads=2, dim=64, vdim=64, chunk=60, rot=64), gated_moe(16, 5, 72, 0.8, 72)),
                             (chunked(heads=5, kv_heads=1, dim=128, vdim=128, chunk=33, rot=96, scale=0.1), gated_moe(4, 2, 64, 0.5, 300, 0.7)),
                             (chunked(heads=20, kv_heads=1, dim=192, vdim=128, chunk=97, rot=128, scale=0.1), None),
                             (chunked(heads=2, kv_heads=2, dim=160, vdim=144, chunk=64, rot=80), gated_moe(8, 8, 160, 1.0, 8))], loop=(2, 4, 2), width=128),
    "chunk of one": desalix([(chunked(heads=2, kv_heads=2, dim=8, vdim=8, chunk=1, rot=8), gated_moe(1, 1, 8, 0.5, 8)),
                             (chunked(heads=9, kv_heads=3, dim=16, vdim=32, chunk=None, rot=4), gated_moe(2, 1, 8, 0.5, None))], loop=(1, 2, 1), width=40),
    "one chunk": desalix([(chunked(chunk=None), gated_moe(shared=None)), (chunked(heads=1, kv_heads=1, dim=8, vdim=8, chunk=128, rot=8), None)]),
    "window of one": config([parallel(heads=20, kv_heads=1, dim=8, vdim=8, window=1, keep=0, rot=8, right_heads=2, right_dim=8)], width=64),
}


def tensors(cfg, seed=0, rank=12):
    """(bfloat16 bit patterns, the same values as float arrays)"""
    bits = stack_models.random_tensors(cfg, seed, rank)
    return bits, {k: stack_models.bits_to_f32(v) for k, v in bits.items()}


def batch(decode, portions, seed=0, extra_pages=5):
    """A batch of decode requests (history lengths) and portions (history, tokens) over permuted pages."""
    return synth.make_batch(decode, portions, vocab=10, seed=seed, extra_pages=extra_pages)


def history_batch(b):
    """The batch that brings every request of b to where b starts, over the same pages (None: all start at zero)."""
    lens = np.diff(b.input_indptr)
    prev = b.kv_len - lens
    reqs = [i for i in range(len(prev)) if prev[i] > 0]
    if not reqs:
        return None, []
    h = synth.make_batch([], [(0, int(prev[i])) for i in reqs], vocab=10, seed=1)
    h.kv_indices = np.concatenate([b.kv_indices[b.kv_indptr[i]:b.kv_indptr[i] + (int(prev[i]) + 15) // 16] for i in reqs]).astype(np.int32)
    return h, reqs
