"""Plain, slow Fesenex: one function per mechanism, float64 numpy on whole
sequences (no cache, no batching, no chunks).  Test oracle only; shares no code
with the product path.

A model is (config, weights): `config` has vocab, width, embedding.scale,
norm.eps and a list of layers (type, mixer sizes, mlp or None); `weights` maps
tensor names to arrays, matrices as [out, in].
"""
import math

import numpy as np


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def embed(weights, tokens, scale):
    return weights["embed"][np.asarray(tokens)] * scale


def distance_bucket(n, rows, far):
    """Row of the distance-bias table for distance n >= 0: exact below half of
    the rows, then logarithmic up to `far`, the last row from there on."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (rows - half)))


def distance_bias(rel, n, far):
    """[heads, query, key]; keys after the query get the row of distance 0."""
    rows = np.array([distance_bucket(d, len(rel), far) for d in range(n)])
    i, j = np.arange(n)[:, None], np.arange(n)[None]
    return np.moveaxis(rel[rows[np.maximum(i - j, 0)]], -1, 0)


def query_temperature(n, coef, every):
    p = np.arange(n)
    return 1.0 + coef * np.log((p + 1) // every + 1.0)


def causal_softmax(scores):
    """scores [heads, query, key] -> weights; query i sees keys 0..i."""
    n = scores.shape[-1]
    s = np.where(np.triu(np.ones((n, n), bool), 1), -np.inf, scores)
    e = np.exp(s - s.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def projection(weights, name, h, heads):
    """[n, heads, size] with the bias"""
    y = h @ weights[name].T + weights[name + ".b"]
    return y.reshape(len(h), heads, -1)


def mix_values(v, first, lam):
    return (1.0 - lam) * v + lam * first


def attention(weights, name, mix, h, eps, first):
    """(output, values): `first` holds the first value-mixing layer's values,
    None in that layer and before it."""
    n, H, G = len(h), mix["heads"], mix["kv_heads"]
    q = rms_norm(projection(weights, name + ".q", h, H), weights[name + ".q.norm"], eps)
    k = rms_norm(projection(weights, name + ".k", h, G), weights[name + ".k.norm"], eps)
    v = projection(weights, name + ".v", h, G)
    if mix.get("q_temp"):
        q = q * query_temperature(n, mix["q_temp"]["coef"], mix["q_temp"]["every"])[:, None, None]
    if mix.get("v_mix") and first is not None:
        v = mix_values(v, first, weights[name + ".vmix"])
    of = np.arange(H) // (H // G)  # each query head's key/value head
    s = np.matmul(q.transpose(1, 0, 2), k[:, of].transpose(1, 2, 0)) * mix["scale"]
    s = s + distance_bias(weights[name + ".rel"], n, mix["bias_max"])
    o = np.matmul(causal_softmax(s), v[:, of].transpose(1, 0, 2))
    return o.transpose(1, 0, 2).reshape(n, -1) @ weights[name + ".o"].T, v


def lightning_states(q, k, v, decay):
    """The recurrence token by token: outputs [n, heads, vdim]."""
    n, H, _ = q.shape
    S = np.zeros((H, q.shape[2], v.shape[2]), q.dtype)
    out = np.empty((n, H, v.shape[2]), q.dtype)
    for t in range(n):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.matmul(q[t][:, None, :], S)[:, 0]
    return out


def lightning(weights, name, mix, h, eps):
    n, H = len(h), mix["heads"]
    q, k, v = (silu(h @ weights[name + s].T).reshape(n, H, -1) for s in (".q", ".k", ".v"))
    o = lightning_states(q, k, v, np.asarray(mix["decay"], h.dtype)).reshape(n, -1)
    o = rms_norm(o, weights[name + ".norm"], eps) * sigmoid(h @ weights[name + ".g"].T)
    return o @ weights[name + ".o"].T


def feed_forward(weights, name, h, limit):
    g = np.minimum(h @ weights[name + ".gate"].T, limit)
    u = np.clip(h @ weights[name + ".up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ weights[name + ".down"].T


def forward(config, weights, tokens, per_layer=None, dtype=np.float64):
    """logits [n, vocab]; per_layer (a list) receives the residual stream
    after every layer."""
    w = {k: np.asarray(v, dtype) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    x = embed(w, tokens, config["embedding"]["scale"])
    first = None
    for i, layer in enumerate(config["layers"]):
        p, mix = "l%d." % i, layer["mixer"]
        h = rms_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "attention":
            y, v = attention(w, p + "mix", mix, h, eps, first)
            if mix.get("v_mix") and first is None:
                first = v
        else:
            y = lightning(w, p + "mix", mix, h, eps)
        x = x + y
        if layer["mlp"] is not None:
            x = x + feed_forward(w, p + "mlp", rms_norm(x, w[p + "norm2"], eps), layer["mlp"]["limit"])
        if per_layer is not None:
            per_layer.append(x.copy())
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T


def greedy(config, weights, prompt, length):
    """(tokens, smallest lead of a pick over the runner-up)"""
    seq, lead = list(prompt), np.inf
    while len(seq) < length:
        z = forward(config, weights, seq)[-1]
        top = np.sort(z)[-2:]
        lead = min(lead, top[1] - top[0])
        seq.append(int(z.argmax()))
    return seq, lead
