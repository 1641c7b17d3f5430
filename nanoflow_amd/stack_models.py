"""Layer-stack designs seen from Python: the tensors a configuration asks for, and random weights of
those shapes (benchmarks, tests, serving without a checkpoint).  What a design computes is known to the
C++ registry (csrc/host/stackModel.h) alone."""
from __future__ import annotations

import json
import os

import numpy as np


def load_config(model) -> dict:
    """A configuration: a dict, a config.json, or the directory that holds one."""
    if isinstance(model, dict):
        return model
    path = os.path.join(model, "config.json") if os.path.isdir(model) else model
    with open(path) as f:
        return json.load(f)


def _zovovik_shapes(cfg: dict, rank: int) -> dict:
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "pos": (cfg["max_positions"], W), "head": (cfg["vocab"], W), "final.norm": (W,)}
    for i, layer in enumerate(cfg["layers"]):
        l, m = f"l{i}.", layer["mixer"]
        out[l + "norm1"] = (W,)
        if layer["type"] == "retention":
            qk, vg = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            out.update({l + "mix.q": (qk, W), l + "mix.k": (qk, W), l + "mix.v": (vg, W), l + "mix.g": (vg, W), l + "mix.o": (W, vg)})
        else:
            a, r = m["left"], m["right"]
            p, q = l + "mix.left.", l + "mix.right."
            out.update({p + "q": (a["heads"] * a["dim"], W), p + "k": (a["kv_heads"] * a["dim"], W),
                        p + "v": (a["kv_heads"] * a["vdim"], W), p + "q.norm": (a["dim"],), p + "k.norm": (a["dim"],),
                        p + "sink": (a["heads"],), p + "o": (W, a["heads"] * a["vdim"])})
            n = r["heads"] * r["dim"]
            out.update({q + "mu." + s: (W,) for s in "rkvgw"})
            out.update({q + s: (n, W) for s in "rkvg"})
            out.update({q + "w1": (rank, W), q + "w2": (n, rank), q + "w0": (n,), q + "u": (r["heads"], r["dim"]),
                        q + "norm": (n,), q + "o": (W, n)})
        if layer.get("mlp"):
            out.update({l + "norm2": (W,), l + "mlp.up": (layer["mlp"]["ff"], W), l + "mlp.down": (W, layer["mlp"]["ff"])})
    return out


def _fipuzen_shapes(cfg: dict, rank: int) -> dict:
    W, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, W), "head": (V, W), "final.norm": (W,), "final.norm.b": (W,)}
    side = (cfg.get("token_side") or {}).get("dim", 0)
    if side:
        out["side.embed"] = (V, side * len(cfg["layers"]))
    for i, layer in enumerate(cfg["layers"]):
        l, x, m = f"l{i}.", f"l{i}.mix.", layer["mixer"]
        out.update({l + "norm1": (W,), l + "norm1.b": (W,)})
        if layer["type"] == "attention":
            for s, n in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                out.update({x + s: (n, W), x + s + ".b": (n,)})
            out.update({x + "g": (m["heads"], W), x + "o": (W, m["heads"] * m["vdim"])})
        elif layer["type"] == "latent_attention":
            H, R = m["heads"], m["kv_rank"]
            out.update({x + "q": (H * (m["dim"] + m["rot_dim"]), W), x + "dkv": (R + m["rot_dim"], W), x + "dkv.norm": (R,),
                        x + "uk": (H * m["dim"], R), x + "uv": (H * m["vdim"], R), x + "o": (W, H * m["vdim"])})
        else:
            qk, vg = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            out.update({x + "q": (qk, W), x + "k": (qk, W), x + "v": (vg, W), x + "g": (vg, W), x + "norm": (vg,), x + "o": (W, vg)})
        if layer.get("mlp"):
            f, r = layer["mlp"]["expert"]["ff"], layer["mlp"]["router"]
            out.update({l + "norm2": (W,), l + "norm2.b": (W,)})
            for e in range(r["experts"]):
                out.update({f"{l}mlp.e{e}.up": (f, W), f"{l}mlp.e{e}.down": (W, f)})
            n = r["experts"] + r.get("identity", 0)
            out.update({l + "mlp.router": (n, W), l + "mlp.correction": (n,)})
        if side:
            out.update({l + "side.gate": (side, W), l + "side.proj": (W, side), l + "side.norm": (W,)})
    return out


def _pudadra_shapes(cfg: dict, rank: int) -> dict:
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "final.norm": (W,)}
    for i, layer in enumerate(cfg["layers"]):
        l, x, m = f"l{i}.", f"l{i}.mix.", layer["mixer"]
        out[l + "norm1"] = (W,)
        if layer["type"] == "attention":
            for s, n in (("q", 2 * m["heads"] * m["dim"]), ("k", 2 * m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                out[x + s] = (n, W)
                if m.get("conv"):
                    out[x + s + ".conv"] = (n, m["conv"])
            out.update({x + s: (m["dim"],) for s in ("lq1", "lk1", "lq2", "lk2")})
        else:
            H, R = m["heads"], m["kv_rank"]
            out.update({x + "q": (H * (m["dim"] + m["rot_dim"]), W), x + "dkv": (R + m["rot_dim"], W), x + "dkv.norm": (R,),
                        x + "uk": (H * m["dim"], R), x + "uv": (H * m["vdim"], R)})
        out[x + "o"] = (W, m["heads"] * m["vdim"])
        f, p = layer.get("mlp"), l + "mlp."
        if not f:
            continue
        out[l + "norm2"] = (W,)
        blocks = {"": f["ff"]} if f["kind"] == "dense" else {f"e{e}.": f["expert"]["ff"] for e in range(f["router"]["experts"])}
        if f["kind"] != "dense":
            out[p + "router"] = (f["router"]["experts"], W)
            if f.get("shared"):
                blocks["shared."] = f["shared"]["ff"]
                out[p + "shared.sg"] = (1, W)
        for b, n in blocks.items():
            out.update({p + b + "up": (n, W), p + b + "down": (W, n)})
    return out


def _desalix_shapes(cfg: dict, rank: int) -> dict:
    W, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, W), "head": (V, W), "final.norm": ()}
    if cfg.get("loop"):
        out["loop.step"] = (cfg["loop"]["times"], W)
    for i, layer in enumerate(cfg["layers"]):
        l, x, m = f"l{i}.", f"l{i}.mix.", layer["mixer"]
        out.update({l + "norm1": (), l + "norm1b": (), l + "ls1": (W,)})
        out.update({x + "q": (m["heads"] * m["dim"], W), x + "k": (m["kv_heads"] * m["dim"], W), x + "v": (m["kv_heads"] * m["vdim"], W),
                    x + "q.norm": (m["dim"],), x + "k.norm": (m["dim"],), x + "sink": (m["heads"],), x + "o": (W, m["heads"] * m["vdim"])})
        f, p = layer.get("mlp"), l + "mlp."
        if not f:
            continue
        out.update({l + "norm2": (), l + "norm2b": (), l + "ls2": (W,), p + "router": (f["router"]["experts"], W)})
        experts = {f"e{e}.": f["expert"]["ff"] for e in range(f["router"]["experts"])}
        if f.get("shared"):
            experts["shared."] = f["shared"]["ff"]
        for e, n in experts.items():
            out.update({p + e + "gate": (n, W), p + e + "up": (n, W), p + e + "down": (W, n)})
    return out


ARCHITECTURES = {"Zovovik": _zovovik_shapes, "Fipuzen": _fipuzen_shapes, "Pudadra": _pudadra_shapes, "Desalix": _desalix_shapes}
# designs whose norms of the residual stream are stored as the difference from one
NORMS_AROUND_ZERO = ("Pudadra",)


def tensor_shapes(cfg: dict, rank: int = 16) -> dict:
    """name -> shape; `rank` is the inner size of the token decay's two-step projection (a tensor's own size, not in
    the configuration)."""
    if cfg.get("architecture") not in ARCHITECTURES:
        raise ValueError(f"unknown architecture {cfg.get('architecture')!r}: one of {', '.join(ARCHITECTURES)}")
    return ARCHITECTURES[cfg["architecture"]](cfg, rank)


def bf16_bits(a) -> np.ndarray:
    """float array -> bfloat16 bit patterns (uint16), round to nearest even."""
    u = np.asarray(a, dtype=np.float32, order="C").view(np.uint32)
    return np.asarray((u + np.uint32(0x7fff) + ((u >> np.uint32(16)) & np.uint32(1))) >> np.uint32(16), dtype=np.uint16)


def bits_to_f32(b) -> np.ndarray:
    return np.asarray(b.astype(np.uint32) << np.uint32(16)).view(np.float32)


def random_tensors(cfg: dict, seed: int = 0, rank: int = 16) -> dict:
    """name -> bfloat16 bit patterns: projections N(0, 1 / inputs), norms around what stands for 1, small biases, shifts in
    [0, 1], token decays that keep a state for a few to a few thousand tokens."""
    rng = np.random.default_rng(seed)
    out, expert_blocks = {}, {}
    for name, shape in tensor_shapes(cfg, rank).items():
        leaf = name.split(".")[-1]
        big = int(np.prod(shape)) > 1 << 22     # large matrices: one block of normals, repeated
        if big and ".mlp.e" in name:            # ... and large experts of a shape share theirs, each from another place on
            if shape not in expert_blocks:
                expert_blocks[shape] = bf16_bits(rng.standard_normal(1 << 22, dtype=np.float32) * shape[-1] ** -0.5)
            out[name] = np.resize(np.roll(expert_blocks[shape], int(rng.integers(1 << 22))), shape)
            continue
        n = min(int(np.prod(shape)), 1 << 22)
        x = rng.standard_normal(n, dtype=np.float32)
        if "norm" in leaf:
            around_zero = cfg["architecture"] in NORMS_AROUND_ZERO and ".mix." not in name
            x = 0.1 * x if around_zero else 1.0 + 0.1 * x
        elif leaf in ("ls1", "ls2"):            # columns count differently, and either way
            x = 0.3 * x + 0.5
        elif leaf in ("lq1", "lk1", "lq2", "lk2"):
            x *= 0.7 * shape[0] ** -0.25
        elif ".mu." in name:
            x = rng.random(n, dtype=np.float32)
        elif leaf == "w0":
            x = -7.0 + 6.0 * rng.random(n, dtype=np.float32)
        elif leaf in ("u", "sink"):
            x = 0.5 * x
        elif leaf == "b":
            x = 0.2 * x
        elif leaf == "correction":
            x = 0.02 * x
        elif name in ("embed", "pos", "side.embed", "loop.step"):
            pass
        else:
            x *= shape[-1] ** -0.5
        b = bf16_bits(x)
        out[name] = (np.resize(b, shape) if big else b.reshape(shape))
    return out


def save_model(directory: str, cfg: dict, tensors: dict):
    """config.json and model.safetensors of `tensors` (bfloat16 bit patterns, float32 or int32 arrays)."""
    os.makedirs(directory, exist_ok=True)
    with open(os.path.join(directory, "config.json"), "w") as f:
        json.dump(cfg, f, indent=1)
    kinds = {np.dtype(np.uint16): "BF16", np.dtype(np.float32): "F32", np.dtype(np.int32): "I32"}
    header, at = {}, 0
    for name, a in tensors.items():
        header[name] = {"dtype": kinds[a.dtype], "shape": list(a.shape), "data_offsets": [at, at + a.nbytes]}
        at += a.nbytes
    h = json.dumps(header).encode()
    h += b" " * (-len(h) % 8)
    with open(os.path.join(directory, "model.safetensors"), "wb") as f:
        f.write(len(h).to_bytes(8, "little") + h)
        for a in tensors.values():
            f.write(np.ascontiguousarray(a).tobytes())
