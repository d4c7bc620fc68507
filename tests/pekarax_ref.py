"""Plain, slow Pekarax: one function per mechanism, float64 numpy on whole
sequences (no cache, no batching, no portions), token by token.  Test oracle only;
shares no code with the product path.

A model is (config, weights): `weights` maps tensor names to arrays, matrices as
[out, in].
"""
import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def soft_cap(z, cap):
    return cap * np.tanh(z / cap)


# ---- norms ----
def unit_rms(x, eps):
    """Every row over its root mean square."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def zero_centred_norm(x, w, eps):
    return unit_rms(x, eps) * (1.0 + w)


def unit_vector(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


# ---- convolution, rotation ----
def causal_conv(u, w):
    """Each channel on its own; the last of `taps` columns meets the current token."""
    taps, out = w.shape[1], np.zeros_like(u)
    for t in range(len(u)):
        for j in range(taps):
            if t - taps + 1 + j >= 0:
                out[t] += w[:, j] * u[t - taps + 1 + j]
    return out


def rotate(x, dims, base):
    """x [T, heads, dim]: columns i and i + dims / 2 turn by p base^(-2 i / dims)."""
    half, out = dims // 2, x.copy()
    for i in range(half):
        a = np.arange(len(x))[:, None] * base ** (-2.0 * i / dims)
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i], out[:, :, i + half] = u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a)
    return out


# ---- mixers: h [T, width] -> [T, width] ----
def attention(h, w, p, c, eps):
    T, H, G = len(h), c["heads"], c["kv_heads"]
    q, k, v = (causal_conv(h @ w[p + n].T, w[p + n + ".conv"]) for n in "qkv")
    q, k, v = q.reshape(T, H, c["dim"]), k.reshape(T, G, c["dim"]), v.reshape(T, G, c["vdim"])
    q, k = (unit_rms(rotate(a, c["rot"]["dims"], c["rot"]["base"]), eps) for a in (q, k))
    out = np.zeros((T, H, c["vdim"]))
    for hd in range(H):
        g = hd // (H // G)
        s = q[:, hd] @ k[:, g].T * c["scale"]
        for t in range(T):
            e = np.exp(s[t, :t + 1] - s[t, :t + 1].max())
            out[t, hd] = e / e.sum() @ v[:t + 1, g]
    return out.reshape(T, -1) @ w[p + "o"].T


def mlstm_read(q, k, v, i, f):
    """Matrix memory of one head: q, k [T, dim], v [T, vdim], log gates i, f [T]."""
    S, n, m, out = np.zeros((k.shape[1], v.shape[1])), np.zeros(k.shape[1]), 0.0, np.zeros(v.shape)
    for t in range(len(q)):
        new = max(f[t] + m, i[t])
        keep, take = np.exp(f[t] + m - new), np.exp(i[t] - new)
        S, n, m = keep * S + take * np.outer(k[t], v[t]), keep * n + take * k[t], new
        out[t] = q[t] @ S / (max(abs(n @ q[t]), np.exp(-m)) + 1e-6)
    return out


def mlstm(h, w, p, c, eps):
    T, H, d, dv, cap = len(h), c["heads"], c["dim"], c["vdim"], c["gate_cap"]
    q = (h @ w[p + "q"].T).reshape(T, H, d) * d ** -0.5
    k, v = (h @ w[p + "k"].T).reshape(T, H, d), (h @ w[p + "v"].T).reshape(T, H, dv)
    i = soft_cap(h @ w[p + "i"].T + w[p + "i.b"], cap)
    f = log_sigmoid(soft_cap(h @ w[p + "f"].T + w[p + "f.b"], cap))
    o = np.stack([unit_rms(mlstm_read(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]), eps) for a in range(H)], 1)
    return (o.reshape(T, -1) * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def gla_read(q, k, v, a):
    """q, k and decays a [T, dim], v [T, vdim]."""
    S, out = np.zeros((k.shape[1], v.shape[1])), np.zeros(v.shape)
    for t in range(len(q)):
        S = a[t][:, None] * S + np.outer(k[t], v[t])
        out[t] = q[t] @ S
    return out


def gla(h, w, p, c, eps):
    T, H, d, dv = len(h), c["heads"], c["dim"], c["vdim"]
    q = (h @ w[p + "q"].T).reshape(T, H, d) * d ** -0.5
    k, v = (h @ w[p + "k"].T).reshape(T, H, d), (h @ w[p + "v"].T).reshape(T, H, dv)
    a = sigmoid(h @ w[p + "a1"].T @ w[p + "a2"].T + w[p + "a2.b"]) ** (1.0 / c["tau"])
    a = a.reshape(T, H, d)
    o = np.stack([unit_rms(gla_read(q[:, i], k[:, i], v[:, i], a[:, i]), eps) * w[p + "norm"] for i in range(H)], 1)
    return (o.reshape(T, -1) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def delta_read(q, k, v, beta, g):
    """q, k and decays g [T, dim], v [T, vdim], beta [T]."""
    S, out = np.zeros((k.shape[1], v.shape[1])), np.zeros(v.shape)
    for t in range(len(q)):
        S = g[t][:, None] * S
        S = S + np.outer(k[t], beta[t] * (v[t] - k[t] @ S))
        out[t] = q[t] @ S
    return out


def channel_delta(h, w, p, c, eps):
    T, H, G, d, dv = len(h), c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    q = unit_vector(q.reshape(T, G, d)) * d ** -0.5
    k, v = unit_vector(k.reshape(T, G, d)), v.reshape(T, H, dv)
    beta = sigmoid(h @ w[p + "b"].T)
    step = softplus(h @ w[p + "a1"].T @ w[p + "a2"].T + w[p + "dt_bias"]).reshape(T, H, d)
    g = np.exp(-np.exp(w[p + "A_log"])[None, :, None] * step)
    gate = sigmoid(h @ w[p + "g1"].T @ w[p + "g2"].T)
    o = [unit_rms(delta_read(q[:, i // (H // G)], k[:, i // (H // G)], v[:, i], beta[:, i], g[:, i]), eps) * w[p + "norm"]
         for i in range(H)]
    return (np.stack(o, 1).reshape(T, -1) * gate) @ w[p + "o"].T


def parallel(h, w, p, c, eps):
    return (c["left_scale"] * attention(h, w, p + "left.", c["left"], eps)
            + c["right_scale"] * mlstm(h, w, p + "right.", c["right"], eps))


MIXERS = {"parallel": parallel, "gla": gla, "channel_delta": channel_delta}


# ---- feed-forward ----
def route(z, correction, r):
    """z [outputs] of one token: the chosen outputs and their weights."""
    s = np.exp(z - z.max())
    s /= s.sum()
    choice = s + correction
    groups = r.get("groups") or {"count": 1, "keep": 1}
    size = len(z) // groups["count"]
    best = sorted(range(groups["count"]), key=lambda i: -choice[i * size:(i + 1) * size].max())[:groups["keep"]]
    allowed = [e for e in range(len(z)) if e // size in best]
    picked = sorted(allowed, key=lambda e: -choice[e])[:r["top"]]
    return picked, s[picked] / (s[picked].sum() + 1e-20) * r["scale"]


def expert(x, w, p, limit):
    g, u = np.minimum(w[p + "gate"] @ x, limit), np.clip(w[p + "up"] @ x, -limit, limit)
    return w[p + "down"] @ (g * sigmoid(1.702 * g) * (u + 1.0))


def experts(h, w, p, c):
    r, out = c["router"], np.zeros_like(h)
    for t, x in enumerate(h):
        for e, wt in zip(*route(w[p + "router"] @ x, w[p + "correction"], r)):
            out[t] += wt * (expert(x, w, p + "e%d." % e, c["expert"]["limit"]) if e < r["experts"] else x)
    return out


# ---- the model ----
def forward(cfg, w, tokens, layers=None):
    """Logits [T, vocab]; layers: a list that takes x after every layer."""
    x, eps, alpha = w["embed"][np.asarray(tokens)], cfg["norm"]["eps"], cfg["postln_alpha"]
    for i, l in enumerate(cfg["layers"]):
        p = "l%d." % i
        x = zero_centred_norm(alpha * x + MIXERS[l["type"]](x, w, p + "mix.", l["mixer"], eps), w[p + "norm1"], eps)
        if l.get("mlp"):
            x = zero_centred_norm(alpha * x + experts(x, w, p + "mlp.", l["mlp"]), w[p + "norm2"], eps)
        if layers is not None:
            layers.append(x)
    return zero_centred_norm(x, w["final.norm"], eps) @ w["head"].T


def greedy(cfg, w, prompt, length):
    """(tokens up to `length`, the smallest lead of a pick over the runner-up)"""
    toks, lead = list(prompt), np.inf
    while len(toks) < length:
        z = np.sort(forward(cfg, w, toks)[-1])
        lead = min(lead, z[-1] - z[-2])
        toks.append(int(forward(cfg, w, toks)[-1].argmax()))
    return toks, lead
