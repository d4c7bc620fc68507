"""Plain, slow Nomutar: one function per mechanism, float64 numpy on whole
sequences (no cache, no batching, no portions).  Test oracle only; shares no
code with the product path.

A model is (config, weights): `weights` maps tensor names to arrays, matrices as
[out, in].
"""
import math

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def soft_cap(z, cap):
    return z if not cap else cap * np.tanh(z / cap)


# ---- embedding ----
def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    t = np.asarray(tokens, np.int64)
    rows = np.full(len(t), buckets, np.int64)  # the last row: no token before
    rows[1:] = (t[:-1] * mul_prev + t[1:] * mul_cur) % buckets
    return rows


def embed(w, tokens, e):
    x = w["embed"][np.asarray(tokens)] * e["scale"]
    if e.get("bigram"):
        b = e["bigram"]
        x = x + w["bigram"][bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"])]
    return x


# ---- norms, convolution ----
def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def group_norm(x, w, eps, groups):
    """RMS norm of each of `groups` equal parts of the vector."""
    parts = x.reshape(len(x), groups, -1)
    return (parts / np.sqrt(np.mean(parts * parts, axis=-1, keepdims=True) + eps)).reshape(x.shape) * w


def causal_conv(h, w):
    """Each channel on its own; tap j of `taps` reads taps - 1 - j tokens back."""
    taps, out = w.shape[1], np.zeros_like(h)
    for j in range(taps):
        back = taps - 1 - j
        out[back:] += w[:, j] * h[:len(h) - back] if back < len(h) else 0.0
    return out


# ---- rotation ----
def inverse_frequencies(dims, base):
    return np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)])


def llama3_frequencies(f, factor, low, high, original):
    out = []
    for v in f:
        wavelength = 2.0 * math.pi / v
        s = (original / wavelength - low) / (high - low)
        out.append(v if wavelength < original / high else v / factor if wavelength > original / low
                   else (1.0 - s) * v / factor + s * v)
    return np.array(out)


def yarn_frequencies(f, dims, base, factor, original, fast, slow):
    """(frequencies, multiplier of cos and sin)"""
    def at(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(at(fast)), 0), min(math.ceil(at(slow)), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / factor * ramp + f * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


def rotate(x, angles, layout, mult=1.0):
    """x [n, heads, size], angles [n, pairs]: the first 2 * pairs elements turn."""
    pairs = angles.shape[1]
    a, b = (np.arange(pairs), np.arange(pairs) + pairs) if layout == "half" else \
           (2 * np.arange(pairs), 2 * np.arange(pairs) + 1)
    c, s = mult * np.cos(angles)[:, None], mult * np.sin(angles)[:, None]
    out = x.copy()
    out[..., a] = x[..., a] * c - x[..., b] * s
    out[..., b] = x[..., b] * c + x[..., a] * s
    return out


# what the mixer's type fixes; the sizes and constants come from the configuration
TYPES = {"attention": dict(norm=True, bias=False, layout="half", scaling="llama3", turn_values=True, sink="learned"),
         "attention_2": dict(norm=False, bias=True, layout="pairs", scaling="yarn", turn_values=False, sink="one"),
         "attention_3": dict(norm=True, bias=False, layout="half", scaling=None, turn_values=False, sink=None)}


def frequencies(rot, kind):
    f, sc = inverse_frequencies(rot["dims"], rot["base"]), rot.get("scaling")
    if kind == "llama3" and sc:
        return llama3_frequencies(f, sc["factor"], sc["low"], sc["high"], sc["original"]), 1.0
    if kind == "yarn" and sc:
        return yarn_frequencies(f, rot["dims"], rot["base"], sc["factor"], sc["original"], sc["fast"], sc["slow"])
    return f, 1.0


# ---- attention ----
def visible(n, size):
    """[query, key]: keys up to the query, the last `size` of them (0: all)"""
    d = np.arange(n)[:, None] - np.arange(n)[None]
    return (d >= 0) & (d < size) if size else d >= 0


def softmax_with_sink(scores, mask, sink):
    """scores [heads, query, key]; sink [heads] or None: one more term below"""
    s = np.where(mask, scores, -np.inf)
    top = s.max(-1, keepdims=True)
    if sink is not None:
        top = np.maximum(top, sink[:, None, None])
    e = np.exp(s - top)
    total = e.sum(-1, keepdims=True)
    if sink is not None:
        total = total + np.exp(sink[:, None, None] - top)
    return e / total


def projection(w, name, h, heads, bias, norm, eps):
    """[n, heads, size]; the norm runs over all heads at once"""
    y = h @ w[name].T
    if bias:
        y = y + w[name + ".b"]
    if norm:
        y = rms_norm(y, w[name + ".norm"], eps)
    return y.reshape(len(h), heads, -1)


def turn_back(o, positions, base, layout):
    f = inverse_frequencies(o.shape[-1], base)
    return rotate(o, -positions[:, None] * f, layout)


def attention(w, name, kind, mix, h, eps):
    t, n, H, G = TYPES[kind], len(h), mix["heads"], mix["kv_heads"]
    q = projection(w, name + ".q", h, H, t["bias"], t["norm"], eps)
    k = projection(w, name + ".k", h, G, t["bias"], t["norm"], eps)
    v = projection(w, name + ".v", h, G, t["bias"], False, eps)
    pos = np.arange(n, dtype=np.float64)
    f, mult = frequencies(mix["rot"], t["scaling"])
    q, k = (rotate(a, pos[:, None] * f, t["layout"], mult) for a in (q, k))
    if t["turn_values"]:
        v = rotate(v, pos[:, None] * inverse_frequencies(mix["vdim"], mix["rot"]["base"]), t["layout"])
    of = np.arange(H) // (H // G)  # each query head's key/value head
    s = np.matmul(q.transpose(1, 0, 2), k[:, of].transpose(1, 2, 0)) * mix["scale"]
    s = soft_cap(s, mix.get("softcap"))
    sink = {"learned": w.get(name + ".sink"), "one": np.zeros(H), None: None}[t["sink"]]
    size = (mix.get("mask") or {}).get("size", 0)
    o = np.matmul(softmax_with_sink(s, visible(n, size), sink), v[:, of].transpose(1, 0, 2)).transpose(1, 0, 2)
    if t["turn_values"]:
        o = turn_back(o, pos, mix["rot"]["base"], t["layout"])
    return o.reshape(n, -1) @ w[name + ".o"].T


# ---- feed-forward ----
def gated(w, name, h):
    return (silu(h @ w[name + ".gate"].T) * (h @ w[name + ".up"].T)) @ w[name + ".down"].T


def route(w, name, h, top):
    """(chosen experts [n, top], their weights)"""
    z = h @ w[name + ".router"].T + w[name + ".router.b"]
    idx = np.argsort(-z, axis=-1, kind="stable")[:, :top]
    c = np.take_along_axis(z, idx, -1)
    e = np.exp(c - c.max(-1, keepdims=True))
    return idx, e / e.sum(-1, keepdims=True)


def shared_gate(w, name, h):
    return sigmoid(h @ w[name + ".shared.sg"].T)


def feed_forward(w, name, mlp, h):
    if mlp["kind"] == "dense":
        return gated(w, name, h)
    idx, wt = route(w, name, h, mlp["router"]["top"])
    y = np.zeros_like(h)
    for t in range(len(h)):
        for e, p in zip(idx[t], wt[t]):
            y[t] += p * gated(w, "%s.e%d" % (name, e), h[t:t + 1])[0]
    if mlp.get("shared"):
        y = y + shared_gate(w, name, h) * gated(w, name + ".shared", h)
    return y


# ---- the model ----
def layer_runs(config):
    """The layers in the order they run: a loop repeats its stretch."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def layer(w, i, cfg, config, x):
    p, eps = "l%d." % i, config["norm"]["eps"]
    h = group_norm(x, w[p + "norm1"], eps, config["norm"]["groups"])
    y = attention(w, p + "mix", cfg["type"], cfg["mixer"], h + causal_conv(h, w[p + "canon1"]), eps)
    if cfg["mlp"] is not None:
        y = y + feed_forward(w, p + "mlp", cfg["mlp"], h)
    return x + config["residual_mult"] * y


def forward(config, weights, tokens, per_layer=None, dtype=np.float64):
    """logits [n, vocab]; per_layer (a list) receives the residual stream
    after every layer run."""
    w = {k: np.asarray(v, dtype) for k, v in weights.items()}
    x = embed(w, tokens, config["embedding"])
    for i in layer_runs(config):
        x = layer(w, i, config["layers"][i], config, x)
        if per_layer is not None:
            per_layer.append(x.copy())
    x = group_norm(x, w["final.norm"], config["norm"]["eps"], config["norm"]["groups"])
    return soft_cap(x @ w["head"].T, config.get("logit_softcap"))


def greedy(config, weights, prompt, length):
    """(tokens, smallest lead of a pick over the runner-up)"""
    seq, lead = list(prompt), np.inf
    while len(seq) < length:
        z = forward(config, weights, seq)[-1]
        top = np.sort(z)[-2:]
        lead = min(lead, top[1] - top[0])
        seq.append(int(z.argmax()))
    return seq, lead
