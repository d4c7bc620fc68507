"""Plain, slow Vapipel: one function per mechanism, float64 numpy on whole
sequences (no cache, no batching).  Test oracle only; shares no code with the
product path.

A model is (config, weights): `config` has vocab, width, max_positions,
norm.eps and a list of layers (type, mixer sizes, mlp or None); `weights` maps
tensor names to arrays [out, in].
"""
import numpy as np


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def embed(weights, tokens):
    n = len(tokens)
    return weights["embed"][np.asarray(tokens)] + weights["pos"][:n]


def latent(weights, name, h, eps):
    """The cached vector of every position: normed down-projection."""
    return rms_norm(h @ weights[name + ".dkv"].T, weights[name + ".dkv.norm"], eps)


def causal_softmax(scores):
    """scores [heads, query, key] -> weights; query i sees keys 0..i."""
    n = scores.shape[-1]
    hidden = np.triu(np.ones((n, n), bool), 1)
    s = np.where(hidden, -np.inf, scores)
    e = np.exp(s - s.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def latent_attention(weights, name, mix, h, c):
    n, H = len(h), mix["heads"]
    q = (h @ weights[name + ".q"].T).reshape(n, H, mix["dim"])
    k = (c @ weights[name + ".uk"].T).reshape(n, H, mix["dim"])
    v = (c @ weights[name + ".uv"].T).reshape(n, H, mix["vdim"])
    p = causal_softmax(np.einsum("ihd,jhd->hij", q, k) * mix["scale"])
    o = np.einsum("hij,jhd->ihd", p, v)
    gate = 1.0 / (1.0 + np.exp(-(h @ weights[name + ".g"].T)))
    return (o * gate[:, :, None]).reshape(n, -1) @ weights[name + ".o"].T


def feed_forward(weights, name, h):
    u = np.maximum(h @ weights[name + ".up"].T, 0.0)
    return (u * u) @ weights[name + ".down"].T


def forward(config, weights, tokens, per_layer=None, dtype=np.float64):
    """logits [n, vocab]; per_layer (a list) receives the residual stream
    after every layer."""
    w = {k: np.asarray(v, dtype) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    x = embed(w, tokens)
    latents = {}
    for i, layer in enumerate(config["layers"]):
        p, mix = "l%d" % i, layer["mixer"]
        src = mix.get("kv_from", i)
        if src == i:
            latents[i] = latent(w, p + ".mix", x, eps)
        x = x + rms_norm(latent_attention(w, p + ".mix", mix, x, latents[src]), w[p + ".norm1"], eps)
        if layer["mlp"] is not None:
            x = x + rms_norm(feed_forward(w, p + ".mlp", x), w[p + ".norm2"], eps)
        if per_layer is not None:
            per_layer.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T


def greedy(config, weights, prompt, length):
    """prompt extended to `length` tokens, and the smallest lead of a pick."""
    seq, lead = list(prompt), np.inf
    while len(seq) < length:
        top = forward(config, weights, seq)[-1]
        order = np.argsort(-top, kind="stable")
        lead = min(lead, top[order[0]] - top[order[1]])
        seq.append(int(order[0]))
    return seq, lead
