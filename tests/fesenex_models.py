"""Small Fesenex models for the tests: configurations and random weights
(values exact in bf16)."""
import numpy as np

from vapipel_models import bf16, write_checkpoint  # noqa: F401


def attention(heads, kv_heads, dim, vdim, scale, bias_max=50, q_temp=None, v_mix=False, ff=None, limit=1.5,
              rel_rows=12):
    """rel_rows: rows of the distance-bias table (a tensor's size, not in the configuration)"""
    mix = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, bias_max=bias_max, v_mix=v_mix)
    if q_temp is not None:
        mix["q_temp"] = dict(coef=q_temp[0], every=q_temp[1])
    return dict(type="attention", mixer=mix, mlp=mlp(ff, limit)), rel_rows


def lightning(heads, dim, vdim, decay, ff=None, limit=1.5):
    return dict(type="lightning", mixer=dict(heads=heads, dim=dim, vdim=vdim, decay=list(decay)),
                mlp=mlp(ff, limit)), None


def mlp(ff, limit):
    return None if ff is None else dict(kind="dense", ff=ff, limit=limit)


def model_config(vocab, width, layers, scale=1.0, eps=1e-5):
    """(configuration, rows of each layer's distance-bias table)"""
    return dict(architecture="Fesenex", vocab=vocab, width=width, embedding=dict(scale=scale),
                norm=dict(eps=eps), layers=[l for l, _ in layers]), [r for _, r in layers]


def shapes(cfg, rel_rows):
    V, W = cfg["vocab"], cfg["width"]
    out = {"embed": (V, W), "final.norm": (W,), "head": (V, W)}
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], "l%d." % i
        H, d, vd = m["heads"], m["dim"], m["vdim"]
        out[p + "norm1"] = (W,)
        if l["type"] == "attention":
            G = m["kv_heads"]
            for n, rows in (("q", H * d), ("k", G * d), ("v", G * vd)):
                out[p + "mix." + n] = (rows, W)
                out[p + "mix." + n + ".b"] = (rows,)
            out[p + "mix.q.norm"] = out[p + "mix.k.norm"] = (d,)
            out[p + "mix.rel"] = (rel_rows[i], H)
            if m["v_mix"]:
                out[p + "mix.vmix"] = ()
        else:
            for n, rows in (("q", H * d), ("k", H * d), ("v", H * vd), ("g", H * vd)):
                out[p + "mix." + n] = (rows, W)
            out[p + "mix.norm"] = (H * vd,)
        out[p + "mix.o"] = (W, H * vd)
        if l["mlp"] is not None:
            ff = l["mlp"]["ff"]
            out[p + "norm2"] = (W,)
            out[p + "mlp.gate"] = out[p + "mlp.up"] = (ff, W)
            out[p + "mlp.down"] = (W, ff)
    return out


def random_weights(model, seed, sharp=1.0):
    """Unit-scale activations; `sharp` multiplies the attention scores."""
    cfg, rel_rows = model
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in shapes(cfg, rel_rows).items():
        if "norm" in name:
            a = 1.0 + 0.3 * rng.standard_normal(shape)
        elif name.endswith("vmix"):
            a = np.asarray(rng.uniform(0.25, 0.75))
        elif name.endswith(".rel"):
            a = 1.5 * rng.standard_normal(shape)
        elif name.endswith(".b"):
            a = 0.4 * rng.standard_normal(shape)
        elif name == "embed":
            a = rng.standard_normal(shape) / cfg["embedding"]["scale"]
        else:
            a = rng.standard_normal(shape) / np.sqrt(shape[1])
        if name.endswith("q.norm"):
            m = cfg["layers"][int(name[1:name.index(".")])]["mixer"]
            a = a * sharp / (m["scale"] * np.sqrt(m["dim"]))
        w[name] = bf16(a).reshape(shape)
    return w
