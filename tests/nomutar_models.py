"""Small Nomutar models for the tests: configurations and random weights (values
exact in bf16)."""
import numpy as np

from vapipel_models import bf16, write_checkpoint  # noqa: F401


def mixer(kind, heads, kv_heads, dim, vdim, scale, rot=None, base=100.0, scaling=None, window=None, cap=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale,
             rot=dict(base=base, dims=dim if rot is None else rot))
    if scaling:
        m["rot"]["scaling"] = dict(scaling)
    if window:
        m["mask"] = dict(size=window)
    if cap:
        m["softcap"] = cap
    return dict(type=kind, mixer=m, mlp=None)


def turned(*a, **kw):
    return mixer("attention", *a, **kw)


def biased(*a, **kw):
    return mixer("attention_2", *a, **kw)


def plain(*a, **kw):
    return mixer("attention_3", *a, **kw)


def dense(layer, ff):
    return dict(layer, mlp=dict(kind="dense", ff=ff))


def experts(layer, n, top, ff, shared=None):
    mlp = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=n, top=top))
    if shared:
        mlp["shared"] = dict(ff=shared)
    return dict(layer, mlp=mlp)


# scalings whose every branch some frequency of the tests' small bases takes
LLAMA3 = dict(factor=4.0, low=1.0, high=4.0, original=64)
YARN = dict(factor=4.0, original=64, fast=8.0, slow=1.0)


def model_config(vocab, width, layers, groups=1, taps=3, mult=0.7, loop=None, cap=None, scale=1.0, eps=1e-5,
                 bigram=(101, 31, 7)):
    c = dict(architecture="Nomutar", vocab=vocab, width=width, embedding=dict(scale=scale),
             norm=dict(eps=eps, groups=groups), canon=dict(taps=taps), residual_mult=mult, layers=layers)
    if bigram:
        c["embedding"]["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    if cap:
        c["logit_softcap"] = cap
    return c


def shapes(cfg):
    V, W = cfg["vocab"], cfg["width"]
    out = {"embed": (V, W), "final.norm": (W,), "head": (V, W)}
    if cfg["embedding"].get("bigram"):
        out["bigram"] = (cfg["embedding"]["bigram"]["buckets"] + 1, W)

    def gated(p, ff):
        out[p + "gate"] = out[p + "up"] = (ff, W)
        out[p + "down"] = (W, ff)

    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], "l%d." % i
        H, G, d, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out[p + "norm1"], out[p + "canon1"] = (W,), (W, cfg["canon"]["taps"])
        for n, rows in (("q", H * d), ("k", G * d), ("v", G * vd)):
            out[p + "mix." + n] = (rows, W)
            if l["type"] == "attention_2":
                out[p + "mix." + n + ".b"] = (rows,)
        if l["type"] != "attention_2":
            out[p + "mix.q.norm"], out[p + "mix.k.norm"] = (H * d,), (G * d,)
        if l["type"] == "attention":
            out[p + "mix.sink"] = (H,)
        out[p + "mix.o"] = (W, H * vd)
        mlp = l["mlp"]
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            gated(p + "mlp.", mlp["ff"])
            continue
        n = mlp["router"]["experts"]
        out[p + "mlp.router"], out[p + "mlp.router.b"] = (n, W), (n,)
        for e in range(n):
            gated(p + "mlp.e%d." % e, mlp["expert"]["ff"])
        if mlp.get("shared"):
            gated(p + "mlp.shared.", mlp["shared"]["ff"])
            out[p + "mlp.shared.sg"] = (1, W)
    return out


def most_experts(cfg):
    return max([l["mlp"]["router"]["experts"] for l in cfg["layers"] if l["mlp"] and l["mlp"]["kind"] == "moe"] + [0])


def random_weights(cfg, seed, sharp=1.0):
    """Unit-scale activations; `sharp` multiplies the attention scores.

    Routers: the first channels, as many as there are experts, hold a shuffle of
    evenly spaced levels per token, which no sublayer writes to; a router mostly
    reads them, so no choice of experts is a close call that rounding turns."""
    rng = np.random.default_rng(seed)
    E, w = most_experts(cfg), {}
    for name, shape in shapes(cfg).items():
        layer = cfg["layers"][int(name[1:name.index(".")])] if name[0] == "l" else None
        if name.endswith("norm") or name.endswith("norm1"):
            a = 1.0 + 0.3 * rng.standard_normal(shape)
            if name.endswith("norm1"):
                a[:E] = 1.0
        elif name.endswith(".b"):
            a = 0.3 * rng.standard_normal(shape) * (0.1 / max(E, 1) if "router" in name else 1.0)
        elif name.endswith("sink"):
            a = 1.0 + rng.standard_normal(shape)
        elif name.endswith("canon1"):
            a = 0.5 * rng.standard_normal(shape)
        elif name == "embed":
            a = rng.standard_normal(shape)
            if E:
                a[:, :E] = np.stack([rng.permutation(np.linspace(-2.0, 2.0, E)) for _ in range(shape[0])])
            a = a / cfg["embedding"]["scale"]
        elif name == "bigram":
            a = 0.7 * rng.standard_normal(shape)
            a[:, :E] = 0.0
        elif name.endswith("router"):
            a = rng.standard_normal(shape) * 0.2 / (max(shape[0], 2) * np.sqrt(shape[1]))
            a[np.arange(shape[0]), rng.permutation(E)[:shape[0]]] += 3.0
        else:
            a = rng.standard_normal(shape) / np.sqrt(shape[1])
            if name.endswith("mix.o") or name.endswith("down"):
                a[:E] = 0.0
        if layer and (name.endswith("q.norm") or (layer["type"] == "attention_2" and name.endswith("mix.q"))):
            a = a * sharp / (layer["mixer"]["scale"] * np.sqrt(layer["mixer"]["dim"]))
        w[name] = bf16(a).reshape(shape)
    return w
