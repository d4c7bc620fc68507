"""Small Pekarax models for the tests: configurations and random weights (values
exact in bf16)."""
import numpy as np

from vapipel_models import bf16, write_checkpoint  # noqa: F401


def delta(heads, kv_heads, dim, vdim, conv=3, low=(7, 5)):
    """low: columns of the two narrow products (a checkpoint's, not the configuration's)"""
    return dict(type="channel_delta", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv), mlp=None,
                low=list(low))


def gla(heads, dim, vdim, tau=4.0, low=6):
    return dict(type="gla", mixer=dict(heads=heads, dim=dim, vdim=vdim, tau=tau), mlp=None, low=[low])


def parallel(left, right, left_scale=0.7, right_scale=0.6):
    """left: (heads, kv_heads, dim, vdim, scale) and optionally rot, base, conv; right: (heads, dim, vdim, cap)"""
    H, G, d, dv, scale, rot, base, conv = tuple(left) + (None, 100.0, 3)[len(left) - 5:]
    a = dict(heads=H, kv_heads=G, dim=d, vdim=dv, scale=scale, conv=conv, rot=dict(base=base, dims=d if rot is None else rot))
    m = dict(zip(("heads", "dim", "vdim", "gate_cap"), right))
    return dict(type="parallel", mixer=dict(left=a, right=m, left_scale=left_scale, right_scale=right_scale), mlp=None)


def experts(layer, n, top, ff, identity=0, groups=None, scale=1.5, limit=0.8):
    r = dict(experts=n, top=top, identity=identity, scale=scale)
    if groups:
        r["groups"] = dict(zip(("count", "keep"), groups))
    return dict(layer, mlp=dict(kind="moe", expert=dict(ff=ff, limit=limit), router=r))


def model_config(vocab, width, layers, alpha=2.5, eps=1e-5):
    return dict(architecture="Pekarax", vocab=vocab, width=width, norm=dict(eps=eps), postln_alpha=alpha, layers=layers)


def outputs(layer):
    r = layer["mlp"]["router"]
    return r["experts"] + r["identity"]


def shapes(cfg):
    V, W = cfg["vocab"], cfg["width"]
    out = {"embed": (V, W), "final.norm": (W,), "head": (V, W)}

    def heads(p, H, G, d, dv, conv=0):
        for n, rows in (("q", G * d if conv < 0 else H * d), ("k", G * d), ("v", (H if conv <= 0 else G) * dv)):
            out[p + n] = (rows, W)
            if conv:
                out[p + n + ".conv"] = (rows, abs(conv))
        out[p + "o"] = (W, H * dv)

    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], "l%d.mix." % i
        out["l%d.norm1" % i] = (W,)
        if l["type"] == "parallel":
            a, r = m["left"], m["right"]
            heads(p + "left.", a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["conv"])
            H, d, dv = r["heads"], r["dim"], r["vdim"]
            heads(p + "right.", H, H, d, dv)
            out[p + "right.g"], out[p + "right.norm"] = (H * dv, W), (H * dv,)
            for n in "if":
                out[p + "right." + n], out[p + "right." + n + ".b"] = (H, W), (H,)
        else:
            H, d, dv = m["heads"], m["dim"], m["vdim"]
            out[p + "norm"] = (dv,)
            out[p + "a1"], out[p + "a2"] = (l["low"][0], W), (H * d, l["low"][0])
            if l["type"] == "gla":
                heads(p, H, H, d, dv)
                out[p + "g"], out[p + "a2.b"] = (H * dv, W), (H * d,)
            else:
                heads(p, H, m["kv_heads"], d, dv, -m["conv"])
                out[p + "g1"], out[p + "g2"] = (l["low"][1], W), (H * dv, l["low"][1])
                out[p + "b"], out[p + "A_log"], out[p + "dt_bias"] = (H, W), (H,), (H * d,)
        if l["mlp"]:
            out["l%d.norm2" % i] = (W,)
            f, n, ff = "l%d.mlp." % i, outputs(l), l["mlp"]["expert"]["ff"]
            out[f + "router"], out[f + "correction"] = (n, W), (n,)
            for e in range(l["mlp"]["router"]["experts"]):
                out[f + "e%d.gate" % e] = out[f + "e%d.up" % e] = (ff, W)
                out[f + "e%d.down" % e] = (W, ff)
    return out


def most_outputs(cfg):
    return max([outputs(l) for l in cfg["layers"] if l["mlp"]] + [0])


def random_weights(cfg, seed):
    """Unit-scale activations.  A memory's keys are partly its queries' rows: a head's
    output goes over its own rms, and where query and keys happen to be orthogonal that
    would blow up rounding.

    Routers: the first channels, as many as there are outputs, hold a shuffle of evenly
    spaced levels per token, which no sublayer writes to; a router mostly reads them, so
    no choice is a close call that rounding turns.  Corrections: one for all, but for
    an expert that is always chosen and one that never is, where there are enough."""
    rng = np.random.default_rng(seed)
    E, w = most_outputs(cfg), {}
    for name, shape in shapes(cfg).items():
        layer = cfg["layers"][int(name[1:name.index(".")])] if name[0] == "l" else None
        if name.endswith(("norm1", "norm2", "final.norm")):
            a = 0.3 * rng.standard_normal(shape)
            if name != "final.norm":
                a[:E] = 0.0
        elif name.endswith("norm"):
            a = 1.0 + 0.3 * rng.standard_normal(shape)
        elif name.endswith("A_log"):
            a = rng.uniform(-3.0, 0.5, shape)
        elif name.endswith("dt_bias"):
            a = rng.uniform(-4.0, 0.0, shape)
        elif name.endswith("a2.b"):
            a = rng.uniform(-1.0, 4.0, shape)
        elif name.endswith("right.i.b"):
            a = rng.uniform(-1.0, 1.0, shape)
        elif name.endswith("right.f.b"):
            a = rng.uniform(1.0, 6.0, shape)
        elif name.endswith("right.i"):
            a = rng.standard_normal(shape) / np.sqrt(shape[1]) * 2.0
        elif name.endswith("correction"):
            a = np.full(shape, -0.7)
            r = layer["mlp"]["router"]
            count, keep = (r.get("groups") or dict(count=1, keep=1)).values()
            room = shape[0] // count * keep
            if shape[0] > 3 and room > r["top"] + 1:
                a[rng.permutation(shape[0])[:2]] += np.array([4.0, -4.0])
        elif name == "embed":
            a = rng.standard_normal(shape)
            if E:
                a[:, :E] = np.stack([rng.permutation(np.linspace(-2.0, 2.0, E)) for _ in range(shape[0])])
        elif name.endswith("router"):
            a = rng.standard_normal(shape) * 0.02 / np.sqrt(shape[1])
            a[np.arange(shape[0]), rng.permutation(E)[:shape[0]]] += max(1.0, 0.15 * (E - 1))
        elif name.endswith("conv"):
            a = rng.standard_normal(shape) / np.sqrt(shape[1])
        else:
            a = rng.standard_normal(shape) / np.sqrt(shape[1])
            if name.endswith((".o", "down")):
                a[:E] = 0.0
            if name.endswith(("mix.k", "right.k")):
                a = 0.8 * w[name[:-1] + "q"] + 0.6 * a
        w[name] = bf16(a).reshape(shape)
    return w
