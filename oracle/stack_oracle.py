"""Plain, slow float64 restatement of the layer-stack designs (decoders put together from a list of
layers).  Zovovik: retention, windowed attention with kept first tokens and a sink, a token-shift recurrence
with data-dependent decay, two mixers side by side.  Fipuzen: attention with a unit sink, a query temperature
and a gate per head, latent attention, lightning attention, a mixture of experts with identity experts, token
inputs to every layer.  Pudadra: differential attention over a window on convolved projections with capped
scores, latent attention over a window, experts in groups of which some are left out, a gated shared
expert.  Desalix: attention in chunks with normed, turned values and a sink, norms on both sides of a sublayer
with one number each, layer scales, a run of layers passed several times, clamped gated experts whose input is
weighed.  Test infrastructure only: one function per mechanism, whole sequences at once, nothing
shared with the product path.

A model is (config, tensors): the parsed config.json and a dict name -> numpy array (any float type).
Nothing is cached between calls and every token sees the whole sequence before it, so this says what
the logits are whatever way a serving engine cuts the tokens up.
"""
from __future__ import annotations

import numpy as np


def f64(a):
    return np.asarray(a, dtype=np.float64)


def rms_norm(x, eps, w=None):
    y = x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)
    return y if w is None else y * f64(w)


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


def squared_relu(z):
    return np.maximum(z, 0.0) ** 2


def rotate(x, positions, dims, base, interleaved):
    """x [T, heads, d]; the first `dims` of d are turned by position * base^(-2i/dims), in pairs
    (i, i + dims/2), or (2i, 2i + 1) when interleaved."""
    if dims == 0:
        return x.copy()
    half = dims // 2
    i = np.arange(half, dtype=np.float64)
    angle = f64(positions)[:, None] * f64(base) ** (-2.0 * i / dims)       # [T, half]
    c, s = np.cos(angle)[:, None, :], np.sin(angle)[:, None, :]
    first, second = (2 * np.arange(half), 2 * np.arange(half) + 1) if interleaved else \
        (np.arange(half), np.arange(half) + half)
    u, v = x[..., first], x[..., second]
    out = x.copy()
    out[..., first] = u * c - v * s
    out[..., second] = v * c + u * s
    return out


def window_mask(T, size, keep_first):
    """[T, T] bool: does position i see position j."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def sink_attention(q, k, v, mask, scale, sink, cap=None):
    """q [T, H, d], k [T, G, d], v [T, G, e], sink [H] (or None): softmax whose denominator also
    holds exp(sink)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = np.empty((T, H, v.shape[-1]))
    for h in range(H):
        s = np.where(mask, capped((q[:, h] @ k[:, h // per].T) * scale, cap), -np.inf)
        m = s.max(axis=1, keepdims=True)
        if sink is not None:
            m = np.maximum(m, f64(sink)[h])
        p = np.exp(s - m)
        den = p.sum(axis=1, keepdims=True)
        if sink is not None:
            den = den + np.exp(f64(sink)[h] - m)
        out[:, h] = (p / den) @ v[:, h // per]
    return out


def fixed_decay_recurrence(q, k, v, decay):
    """Per head: the state fades by a constant, takes in key (x) value, and is then read by the query."""
    T, H, d = q.shape
    S = np.zeros((H, d, v.shape[-1]))
    out = np.empty((T, H, v.shape[-1]))
    g = f64(decay)[:, None, None]
    for t in range(T):
        S = g * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hkv,hk->hv", S, q[t])
    return out


def bonus_recurrence(r, k, v, w, u):
    """Per head: the state is read first, with the current key weighted by u; then each of its rows fades
    by the token's own factor and takes in key (x) value."""
    T, H, d = r.shape
    S = np.zeros((H, d, v.shape[-1]))
    out = np.empty((T, H, v.shape[-1]))
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hkv,hk->hv", S + f64(u)[:, :, None] * kv, r[t])
        S = w[t][:, :, None] * S + kv
    return out


def previous_token(h):
    return np.concatenate([np.zeros_like(h[:1]), h[:-1]], axis=0)


def linear(t, name, x):
    return x @ f64(t[name]).T


def retention_mixer(t, pre, m, eps, h, positions):
    T, H = h.shape[0], m["heads"]
    q = linear(t, pre + "q", h).reshape(T, H, m["dim"])
    k = linear(t, pre + "k", h).reshape(T, H, m["dim"])
    v = linear(t, pre + "v", h).reshape(T, H, m["vdim"])
    rot = m["rot"]
    q = rotate(q, positions, rot["dims"], rot["base"], False)
    k = rotate(k, positions, rot["dims"], rot["base"], False) * m["dim"] ** -0.5
    o = rms_norm(fixed_decay_recurrence(q, k, v, m["decay"]), eps).reshape(T, -1)
    return linear(t, pre + "o", o * silu(linear(t, pre + "g", h)))


def window_attention_mixer(t, pre, m, eps, h, positions):
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = linear(t, pre + "q", h).reshape(T, H, m["dim"])
    k = linear(t, pre + "k", h).reshape(T, G, m["dim"])
    v = linear(t, pre + "v", h).reshape(T, G, m["vdim"])
    rot = m["rot"]
    q = rotate(rms_norm(q, eps, t[pre + "q.norm"]), positions, rot["dims"], rot["base"], True)
    k = rotate(rms_norm(k, eps, t[pre + "k.norm"]), positions, rot["dims"], rot["base"], True)
    mask = window_mask(T, m["mask"]["size"], m["mask"]["keep_first"])
    o = sink_attention(q, k, v, mask, m["scale"], t[pre + "sink"])
    return linear(t, pre + "o", o.reshape(T, -1))


def token_shift_mixer(t, pre, m, eps, h):
    T, H, d = h.shape[0], m["heads"], m["dim"]
    prev = previous_token(h)
    mix = {s: h + (prev - h) * f64(t[pre + "mu." + s]) for s in "rkvgw"}
    r, k, v = (linear(t, pre + s, mix[s]).reshape(T, H, d) for s in "rkv")
    gate = silu(linear(t, pre + "g", mix["g"]))
    z = linear(t, pre + "w2", np.tanh(linear(t, pre + "w1", mix["w"]))) + f64(t[pre + "w0"])
    w = np.exp(-np.exp(z)).reshape(T, H, d)
    o = rms_norm(bonus_recurrence(r, k, v, w, t[pre + "u"]), eps).reshape(T, -1)
    return linear(t, pre + "o", o * f64(t[pre + "norm"]) * gate)


def mixer(t, pre, kind, m, eps, h, positions):
    if kind == "retention":
        return retention_mixer(t, pre, m, eps, h, positions)
    assert kind == "parallel", kind
    return (m["left_scale"] * window_attention_mixer(t, pre + "left.", m["left"], eps, h, positions)
            + m["right_scale"] * token_shift_mixer(t, pre + "right.", m["right"], eps, h))


def feed_forward(t, pre, m, h):
    assert m["kind"] == "dense", m
    return linear(t, pre + "down", squared_relu(linear(t, pre + "up", h)))


# ---------------------------------------------------------------- Fipuzen

def layer_norm(x, eps, w, b):
    c = x - x.mean(axis=-1, keepdims=True)
    return c / np.sqrt((c * c).mean(axis=-1, keepdims=True) + eps) * f64(w) + f64(b)


def gelu_erf(z):
    from scipy.special import erf
    return 0.5 * z * (1.0 + erf(z / np.sqrt(2.0)))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def softmax(z):
    e = np.exp(z - z.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def query_temperature(positions, coef, every):
    """Factor of a query at each position; grows with the logarithm of the block of `every` positions it is in."""
    return 1.0 + coef * np.log(np.floor((f64(positions) + 1.0) / every) + 1.0)


def biased_linear(t, name, x):
    return linear(t, name, x) + f64(t[name + ".b"])


def gated_attention_mixer(t, pre, m, h, positions):
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = biased_linear(t, pre + "q", h).reshape(T, H, m["dim"])
    k = biased_linear(t, pre + "k", h).reshape(T, G, m["dim"])
    v = biased_linear(t, pre + "v", h).reshape(T, G, m["vdim"])
    if m.get("q_temp"):
        q = q * query_temperature(positions, m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None]
    o = sink_attention(q, k, v, window_mask(T, T + 1, 0), m["scale"], np.zeros(H))
    o = o * sigmoid(linear(t, pre + "g", h))[:, :, None]
    return linear(t, pre + "o", o.reshape(T, -1))


def lightning_mixer(t, pre, m, eps, h):
    T, H = h.shape[0], m["heads"]
    q, k, v = (silu(linear(t, pre + s, h)).reshape(T, H, -1) for s in "qkv")
    o = fixed_decay_recurrence(q, k, v, m["decay"]).reshape(T, -1)
    return linear(t, pre + "o", rms_norm(o, eps, t[pre + "norm"]) * sigmoid(linear(t, pre + "g", h)))


def latent_attention(q_plain, q_turned, latent, k_turned, w_uk, w_uv, scale, mask=None):
    """q_plain [T, H, d], q_turned [T, H, r], latent [T, c], k_turned [T, r], w_uk [H, d, c], w_uv [H, e, c]: keys and
    values of every head are written out and attended to one head at a time."""
    T, H, _ = q_plain.shape
    mask = window_mask(T, T + 1, 0) if mask is None else mask
    out = np.empty((T, H, w_uv.shape[1]))
    for h in range(H):
        k, v = latent @ w_uk[h].T, latent @ w_uv[h].T
        s = np.where(mask, (q_plain[:, h] @ k.T + q_turned[:, h] @ k_turned.T) * scale, -np.inf)
        out[:, h] = softmax(s) @ v
    return out


def latent_attention_mixer(t, pre, m, eps, h, positions):
    T, H, d, r, c = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    q = linear(t, pre + "q", h).reshape(T, H, d + r)
    down = linear(t, pre + "dkv", h)
    latent = rms_norm(down[:, :c], eps, t[pre + "dkv.norm"])
    turn = lambda x: rotate(x, positions, r, m["rot"]["base"], True)
    o = latent_attention(q[..., :d], turn(q[..., d:]), latent, turn(down[:, None, c:])[:, 0], f64(t[pre + "uk"]).reshape(H, d, c),
                         f64(t[pre + "uv"]).reshape(H, -1, c), m["scale"])
    return linear(t, pre + "o", o.reshape(T, -1))


def route(z, correction, top, scale):
    """(chosen [T, top], weights [T, top]) from router logits."""
    s = softmax(z)
    chosen = np.argsort(-(s + f64(correction)), axis=-1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, axis=-1) * scale


def mixture(t, pre, m, h):
    r = m["router"]
    chosen, weights = route(linear(t, pre + "router", h), t[pre + "correction"], r["top"], r["scale"])
    y = np.zeros_like(h)
    for token in range(h.shape[0]):
        for e, w in zip(chosen[token], weights[token]):
            if e < r["experts"]:
                out = linear(t, f"{pre}e{e}.down", gelu_erf(linear(t, f"{pre}e{e}.up", h[token])))
            else:
                out = h[token]
            y[token] += w * out
    return y


def token_side_input(t, pre, dim, index, eps, x, tokens):
    """What layer `index` adds for the tokens themselves: their own slice of a table, let through by the residual."""
    e = f64(t["side.embed"])[tokens][:, index * dim:(index + 1) * dim]
    y = linear(t, pre + "side.proj", gelu_tanh(linear(t, pre + "side.gate", x)) * e)
    return rms_norm(y, eps, t[pre + "side.norm"])


def fipuzen_forward(cfg, t, tokens, want_layers=False):
    tokens = np.asarray(tokens)
    positions, eps = np.arange(len(tokens)), cfg["norm"]["eps"]
    norm = lambda x, name: layer_norm(x, eps, t[name], t[name + ".b"])
    x = f64(t["embed"])[tokens]
    layers = []
    for i, layer in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", layer["mixer"]
        h = norm(x, pre + "norm1")
        if layer["type"] == "attention":
            x = x + gated_attention_mixer(t, pre + "mix.", m, h, positions)
        elif layer["type"] == "latent_attention":
            x = x + latent_attention_mixer(t, pre + "mix.", m, eps, h, positions)
        else:
            assert layer["type"] == "lightning", layer
            x = x + lightning_mixer(t, pre + "mix.", m, eps, h)
        if layer.get("mlp"):
            x = x + mixture(t, pre + "mlp.", layer["mlp"], norm(x, pre + "norm2"))
        if cfg.get("token_side"):
            x = x + token_side_input(t, pre, cfg["token_side"]["dim"], i, eps, x, tokens)
        layers.append(x)
    logits = linear(t, "head", norm(x, "final.norm"))
    return (logits, np.stack(layers)) if want_layers else logits


# ---------------------------------------------------------------- Pudadra

def short_conv(u, w):
    """u [T, C], w [C, taps]: every channel is mixed over time with the taps - 1 values before it, zeros before the first."""
    T, taps = u.shape[0], w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, u.shape[1])), u])
    return sum(padded[j:j + T] * f64(w)[:, j] for j in range(taps))


def stretched_frequencies(f, factor, low, high, original):
    """Frequencies whose wavelength is short against `original` positions stay, long ones are divided by `factor`, and
    in between one goes over into the other."""
    turns = original * f / (2 * np.pi)          # original / wavelength
    s = np.clip((turns - low) / (high - low), 0.0, 1.0)
    return np.where(turns > high, f, np.where(turns < low, f / factor, (1 - s) * f / factor + s * f))


def rotate_by(x, angles):
    """x [T, heads, d], angles [T, n]: dimensions i and i + n are turned by angle i, those from 2n on stay."""
    n = angles.shape[1]
    c, s = np.cos(angles)[:, None, :], np.sin(angles)[:, None, :]
    u, v = x[..., :n], x[..., n:2 * n]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., 2 * n:]], axis=-1)


def capped(s, cap):
    return s if cap is None else cap * np.tanh(s / cap)


def map_weight(lq1, lk1, lq2, lk2, diff):
    return np.exp(f64(lq1) @ f64(lk1)) - np.exp(f64(lq2) @ f64(lk2)) + diff


def differential_attention(q, k, v, mask, scale, cap, weight, diff, eps):
    """q [T, H, 2, d], k [T, G, 2, d], v [T, G, e]: two attentions over the same values, the second taken off `weight`
    times, and what is left normed per head."""
    T, H = q.shape[:2]
    per = H // k.shape[1]
    out = np.empty((T, H, v.shape[-1]))
    for h in range(H):
        g = h // per
        a = [softmax(np.where(mask, capped((q[:, h, x] @ k[:, g, x].T) * scale, cap), -np.inf)) @ v[:, g] for x in (0, 1)]
        out[:, h] = rms_norm(a[0] - weight * a[1], eps) * (1.0 - diff)
    return out


def differential_attention_mixer(t, pre, m, eps, h, positions):
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k, v = (short_conv(linear(t, pre + s, h), t[pre + s + ".conv"]) for s in "qkv")
    rot = m["rot"]
    f = f64(rot["base"]) ** (-2.0 * np.arange(rot["dims"] // 2) / max(rot["dims"], 1))
    if rot.get("scaling"):
        f = stretched_frequencies(f, **rot["scaling"])
    angles = f64(positions)[:, None] * f
    turn = lambda x, n: rotate_by(x.reshape(T, n * 2, d), angles).reshape(T, n, 2, d)
    weight = map_weight(*(t[pre + s] for s in ("lq1", "lk1", "lq2", "lk2")), m["diff"])
    o = differential_attention(turn(q, H), turn(k, G), v.reshape(T, G, m["vdim"]), window_mask(T, m["mask"]["size"], 0), m["scale"],
                               m.get("softcap"), weight, m["diff"], eps)
    return linear(t, pre + "o", o.reshape(T, -1))


def windowed_latent_attention_mixer(t, pre, m, eps, h, positions):
    T, H, d, r, c = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    q = linear(t, pre + "q", h).reshape(T, H, d + r)
    down = linear(t, pre + "dkv", h)
    latent = rms_norm(down[:, :c], eps, t[pre + "dkv.norm"])
    turn = lambda x: rotate(x, positions, r, m["rot"]["base"], True)
    o = latent_attention(q[..., :d], turn(q[..., d:]), latent, turn(down[:, None, c:])[:, 0], f64(t[pre + "uk"]).reshape(H, d, c),
                         f64(t[pre + "uv"]).reshape(H, -1, c), m["scale"], window_mask(T, m["mask"]["size"], 0))
    return linear(t, pre + "o", o.reshape(T, -1))


def grouped_choice(s, top, count, keep):
    """The `top` largest of s [T, outputs] among the `keep` of `count` runs of neighbours whose largest entries are largest."""
    T, n = s.shape
    best = s.reshape(T, count, n // count).max(axis=-1)
    kept = np.argsort(-best, axis=-1, kind="stable")[:, :keep]
    open_ = np.zeros((T, count), bool)
    np.put_along_axis(open_, kept, True, axis=1)
    return np.argsort(np.where(np.repeat(open_, n // count, axis=1), -s, np.inf), axis=-1, kind="stable")[:, :top]


def shared_expert(t, pre, h):
    y = linear(t, pre + "down", squared_relu(linear(t, pre + "up", h)))
    return sigmoid(linear(t, pre + "sg", h)) * y


def grouped_mixture(t, pre, m, h):
    r = m["router"]
    s = softmax(linear(t, pre + "router", h))
    g = r.get("groups") or {"count": 1, "keep": 1}
    chosen = grouped_choice(s, r["top"], g["count"], g["keep"])
    y = shared_expert(t, pre + "shared.", h) if m.get("shared") else np.zeros_like(h)
    for token in range(h.shape[0]):
        for e in chosen[token]:
            y[token] += s[token, e] * linear(t, f"{pre}e{e}.down", squared_relu(linear(t, f"{pre}e{e}.up", h[token])))
    return y


def pudadra_forward(cfg, t, tokens, want_layers=False):
    tokens = np.asarray(tokens)
    positions, eps, mult = np.arange(len(tokens)), cfg["norm"]["eps"], cfg["residual_mult"]
    norm = lambda x, name: rms_norm(x, eps, 1.0 + f64(t[name]))
    x = f64(t["embed"])[tokens]
    layers = []
    for i, layer in enumerate(cfg["layers"]):
        pre, m, f = f"l{i}.", layer["mixer"], layer.get("mlp")
        mix = {"attention": differential_attention_mixer, "latent_attention": windowed_latent_attention_mixer}[layer["type"]]
        x = x + mult * mix(t, pre + "mix.", m, eps, norm(x, pre + "norm1"), positions)
        if f:
            h = norm(x, pre + "norm2")
            if f["kind"] == "dense":
                x = x + mult * linear(t, pre + "mlp.down", gelu_erf(linear(t, pre + "mlp.up", h)))
            else:
                x = x + mult * grouped_mixture(t, pre + "mlp.", f, h)
        layers.append(x)
    logits = linear(t, "embed", norm(x, "final.norm")) * cfg["logit_scale"]
    return (logits, np.stack(layers)) if want_layers else logits


# ---------------------------------------------------------------- Desalix

def chunk_mask(T, size):
    """[T, T] bool: a position sees those before it in its own run of `size` positions (None: all before it)."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & ((i // size == j // size) if size else True)


def turn_values(v, positions, base, back=False):
    """v [T, heads, e]: all dimensions turned by the position, or back by it."""
    e = v.shape[-1]
    angles = f64(positions)[:, None] * f64(base) ** (-2.0 * np.arange(e // 2) / e)
    return rotate_by(v, -angles if back else angles)


def chunked_attention_mixer(t, pre, m, eps, h, positions):
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    rot = m["rot"]
    q = rms_norm(linear(t, pre + "q", h).reshape(T, H, m["dim"]), eps, t[pre + "q.norm"])
    k = rms_norm(linear(t, pre + "k", h).reshape(T, G, m["dim"]), eps, t[pre + "k.norm"])
    v = rms_norm(linear(t, pre + "v", h).reshape(T, G, m["vdim"]), eps)
    q, k = (rotate(x, positions, rot["dims"], rot["base"], False) for x in (q, k))
    o = sink_attention(q, k, turn_values(v, positions, rot["base"]), chunk_mask(T, (m.get("mask") or {}).get("size")), m["scale"], t[pre + "sink"])
    return linear(t, pre + "o", turn_values(o, positions, rot["base"], back=True).reshape(T, -1))


def clamped_expert(t, pre, limit, h):
    """Gate and up bounded by `limit` (the gate from above only), the gate's sigmoid at 1.702 times itself, one added to up."""
    g = np.minimum(linear(t, pre + "gate", h), limit)
    u = np.clip(linear(t, pre + "up", h), -limit, limit)
    return linear(t, pre + "down", g * sigmoid(1.702 * g) * (u + 1.0))


def sigmoid_choice(z, top):
    """(chosen [T, top], scores [T, top]): every output's own sigmoid, the largest of them as they are."""
    s = sigmoid(z)
    chosen = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, axis=-1)


def input_weighted_mixture(t, pre, m, h):
    chosen, weights = sigmoid_choice(linear(t, pre + "router", h), m["router"]["top"])
    y = clamped_expert(t, pre + "shared.", m["shared"]["limit"], h) if m.get("shared") else np.zeros_like(h)
    for token in range(h.shape[0]):
        for e, w in zip(chosen[token], weights[token]):
            y[token] += clamped_expert(t, f"{pre}e{e}.", m["expert"]["limit"], w * h[token])
    return y


def layer_runs(layers, loop):
    """(layer, number of the pass that starts with it or None), in the order they are run."""
    start, stop, times = (loop["start"], loop["stop"], loop["times"]) if loop else (0, 0, 0)
    runs = [(i, None) for i in range(start)]
    for p in range(times):
        runs += [(i, p if i == start else None) for i in range(start, stop)]
    return runs + [(i, None) for i in range(stop, layers)]


def desalix_forward(cfg, t, tokens, want_layers=False):
    tokens = np.asarray(tokens)
    positions, eps = np.arange(len(tokens)), cfg["norm"]["eps"]
    norm = lambda x, name: rms_norm(x, eps) * float(f64(t[name]).reshape(()))
    embedded = f64(t["embed"])[tokens] * cfg["embedding"]["scale"]
    x, layers = embedded, []
    for i, enters in layer_runs(len(cfg["layers"]), cfg.get("loop")):
        layer, pre = cfg["layers"][i], f"l{i}."
        if enters is not None:
            x = x + (embedded if enters > 0 else 0.0) + f64(t["loop.step"])[enters]
        y = chunked_attention_mixer(t, pre + "mix.", layer["mixer"], eps, norm(x, pre + "norm1"), positions)
        x = x + norm(y, pre + "norm1b") * f64(t[pre + "ls1"])
        if layer.get("mlp"):
            y = input_weighted_mixture(t, pre + "mlp.", layer["mlp"], norm(x, pre + "norm2"))
            x = x + norm(y, pre + "norm2b") * f64(t[pre + "ls2"])
        layers.append(x)
    logits = linear(t, "head", norm(x, "final.norm"))
    return (logits, np.stack(layers)) if want_layers else logits


def forward(cfg, t, tokens, want_layers=False):
    """Logits [T, vocab] of a whole sequence (and the residual stream after every layer)."""
    if cfg["architecture"] == "Fipuzen":
        return fipuzen_forward(cfg, t, tokens, want_layers)
    if cfg["architecture"] == "Pudadra":
        return pudadra_forward(cfg, t, tokens, want_layers)
    if cfg["architecture"] == "Desalix":
        return desalix_forward(cfg, t, tokens, want_layers)
    tokens = np.asarray(tokens)
    positions = np.arange(len(tokens))
    eps = cfg["norm"]["eps"]
    x = f64(t["embed"])[tokens] + f64(t["pos"])[positions]
    layers = []
    for i, layer in enumerate(cfg["layers"]):
        pre = f"l{i}."
        x = x + rms_norm(mixer(t, pre + "mix.", layer["type"], layer["mixer"], eps, x, positions), eps, t[pre + "norm1"])
        if layer.get("mlp"):
            x = x + rms_norm(feed_forward(t, pre + "mlp.", layer["mlp"], x), eps, t[pre + "norm2"])
        layers.append(x)
    logits = linear(t, "head", rms_norm(x, eps, t["final.norm"]))
    return (logits, np.stack(layers)) if want_layers else logits
