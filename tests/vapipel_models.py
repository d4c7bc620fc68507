"""Small Vapipel models for the tests: configurations, random weights (values
exact in bf16) and a checkpoint writer."""
import json
import os
import struct

import numpy as np


def bf16_bits(a):
    b = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((b + 0x7FFF + ((b >> 16) & 1)) >> 16).astype(np.uint16)


def bf16(a):
    """a rounded to bf16, as float32."""
    return (bf16_bits(a).astype(np.uint32) << 16).view(np.float32)


def layer(heads, dim, vdim, kv_rank, scale, ff, kv_from=None):
    mix = dict(heads=heads, dim=dim, vdim=vdim, kv_rank=kv_rank, scale=scale)
    if kv_from is not None:
        mix["kv_from"] = kv_from
    return dict(type="latent_attention", mixer=mix, mlp=None if ff is None else dict(kind="dense", ff=ff))


def model_config(vocab, width, positions, layers, eps=1e-5):
    return dict(architecture="Vapipel", vocab=vocab, width=width, max_positions=positions,
                norm=dict(eps=eps), layers=layers)


def shapes(cfg):
    V, W = cfg["vocab"], cfg["width"]
    out = {"embed": (V, W), "pos": (cfg["max_positions"], W), "final.norm": (W,), "head": (V, W)}
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], "l%d." % i
        H = m["heads"]
        out[p + "norm1"] = (W,)
        out[p + "mix.q"] = (H * m["dim"], W)
        if m.get("kv_from", i) == i:
            out[p + "mix.dkv"] = (m["kv_rank"], W)
            out[p + "mix.dkv.norm"] = (m["kv_rank"],)
        out[p + "mix.uk"] = (H * m["dim"], m["kv_rank"])
        out[p + "mix.uv"] = (H * m["vdim"], m["kv_rank"])
        out[p + "mix.g"] = (H, W)
        out[p + "mix.o"] = (W, H * m["vdim"])
        if l["mlp"] is not None:
            out[p + "norm2"] = (W,)
            out[p + "mlp.up"] = (l["mlp"]["ff"], W)
            out[p + "mlp.down"] = (W, l["mlp"]["ff"])
    return out


def random_weights(cfg, seed, sharp=1.0):
    """Unit-scale activations; `sharp` multiplies the attention scores."""
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in shapes(cfg).items():
        if name.endswith("norm") or name.endswith("norm1") or name.endswith("norm2"):
            a = 1.0 + 0.3 * rng.standard_normal(shape)
        elif name in ("embed", "pos"):
            a = rng.standard_normal(shape) * (1.0 if name == "embed" else 0.5)
        else:
            a = rng.standard_normal(shape) / np.sqrt(shape[1])
        if name.endswith(".uk"):
            m = cfg["layers"][int(name[1:name.index(".")])]["mixer"]
            a *= sharp / (m["scale"] * np.sqrt(m["dim"]))
        w[name] = bf16(a)
    return w


def write_checkpoint(folder, cfg, weights):
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, blobs, off = {}, [], 0
    for name, a in weights.items():
        b = bf16_bits(a).tobytes()
        head[name] = dict(dtype="BF16", shape=list(a.shape), data_offsets=[off, off + len(b)])
        blobs.append(b)
        off += len(b)
    h = json.dumps(head).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(blobs))
    return str(folder)
