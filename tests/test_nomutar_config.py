"""Nomutar configurations and checkpoints: what the reader takes and refuses (no
GPU: a valid configuration ends at the missing device), and the plain
implementation itself."""
import copy
import ctypes

import numpy as np
import pytest

import flexflow_amd as fa
import flexflow_amd.ffmi as F
import nomutar_models as NM
import nomutar_ref as R

CFG = NM.model_config(61, 48, [
    NM.dense(NM.turned(4, 2, 16, 8, 0.3, rot=8, scaling=NM.LLAMA3, window=3, cap=4.0), 40),
    NM.experts(NM.biased(2, 1, 16, 12, 0.2, scaling=NM.YARN, cap=9.0, window=5), 5, 2, 24, shared=16),
    NM.plain(2, 2, 12, 8, 0.2)], groups=3, loop=(0, 2, 2), cap=8.0)
NO_GPU = "no gfx950 device"


def refusal(cfg, **kw):
    with pytest.raises(F.FFMIError) as e:
        fa.Model(cfg, kw.pop("mode", "inc"), max_requests=2, max_tokens=16, max_seq_len=64,
                 max_tree_tokens=0, **kw)
    return str(e.value)


def edited(f):
    c = copy.deepcopy(CFG)
    f(c)
    return c


def no_gpu():
    n = ctypes.c_int(0)
    from hip_util import hip
    return hip().hipGetDeviceCount(ctypes.byref(n)) != 0 or n.value == 0


@pytest.mark.skipif(not no_gpu(), reason="the missing device is the expected end")
@pytest.mark.parametrize("edit", [
    lambda c: None,
    lambda c: c.pop("loop"),
    lambda c: c.update(loop=None),
    lambda c: c.update(loop=dict(start=1, stop=1, times=4)),
    lambda c: c.pop("logit_softcap"),
    lambda c: c["norm"].pop("groups"),
    lambda c: c["embedding"].pop("bigram"),
    lambda c: c["canon"].update(taps=1),
    lambda c: c["layers"][0]["mixer"].pop("mask"),
    lambda c: c["layers"][0]["mixer"].pop("softcap"),
    lambda c: c["layers"][0]["mixer"]["rot"].pop("scaling"),
    lambda c: c["layers"][1]["mixer"]["rot"].update(scaling=None),
    lambda c: c["layers"][1]["mlp"].pop("shared"),
    lambda c: c["layers"][1]["mlp"]["router"].update(top=5),
    lambda c: c.update(layers=c["layers"][2:], loop=None),
])
def test_valid_configurations_reach_the_device_check(edit):
    assert NO_GPU in refusal(edited(edit))
    assert NO_GPU in refusal(edited(edit), full_precision=True)


@pytest.mark.parametrize("edit,what", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c.pop("norm"), "norm.eps"),
    (lambda c: c["norm"].update(groups=5), "norm.groups"),
    (lambda c: c.pop("residual_mult"), "residual_mult"),
    (lambda c: c.pop("canon"), "canon.taps"),
    (lambda c: c["canon"].update(taps=0), "canon.taps"),
    (lambda c: c.update(logit_softcap=0.0), "logit_softcap"),
    (lambda c: c["embedding"].pop("scale"), "embedding.scale"),
    (lambda c: c["embedding"]["bigram"].pop("mul_prev"), "embedding.bigram"),
    (lambda c: c["embedding"]["bigram"].update(mul_cur=0.5), "embedding.bigram"),
    (lambda c: c.update(loop=dict(start=2, stop=1, times=1)), "loop"),
    (lambda c: c.update(loop=dict(start=0, stop=4, times=1)), "loop"),
    (lambda c: c.update(loop=dict(start=0, stop=2, times=0)), "loop"),
    (lambda c: c.update(layers=[]), "layers"),
    (lambda c: c["layers"][0].update(type="attention_9"), "attention_9"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "layers[0].mixer"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "layers[0].mixer"),
    (lambda c: c["layers"][0]["mixer"].update(vdim=7), "layers[0].mixer"),
    (lambda c: c["layers"][0]["mixer"].update(mask=dict(size=0)), "layers[0].mixer.mask"),
    (lambda c: c["layers"][0]["mixer"].update(softcap=-1.0), "layers[0].mixer.softcap"),
    (lambda c: c["layers"][0]["mixer"].pop("rot"), "layers[0].mixer.rot"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "layers[0].mixer.rot"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("high"), "layers[0].mixer.rot.scaling"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].pop("fast"), "layers[1].mixer.rot.scaling"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "layers[0].mlp.kind 'sparse'"),
    (lambda c: c["layers"][0]["mlp"].pop("ff"), "layers[0].mlp"),
    (lambda c: c["layers"][1]["mlp"].pop("expert"), "layers[1].mlp.expert"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=6), "layers[1].mlp.router"),
    (lambda c: c["layers"][1]["mlp"]["shared"].update(ff=0), "layers[1].mlp.shared"),
])
def test_refused_configurations_name_the_place(edit, what):
    assert what in refusal(edited(edit))


def test_tree_and_beam_modes_are_not_offered():
    assert "unsupported" in refusal(CFG, mode="tree")


def test_load_config(tmp_path):
    NM.write_checkpoint(tmp_path, CFG, NM.random_weights(CFG, 1))
    assert fa.load_config(str(tmp_path)) == CFG


# ---- the plain implementation ----
def test_oracle_decodes_as_it_prefills():
    """A longer sequence leaves the earlier positions' logits alone, and every
    tensor that a sequence of this length reaches moves them."""
    w = NM.random_weights(CFG, 2, sharp=3.0)
    toks = [7, 3, 60, 0, 11, 11, 4, 33, 20, 58, 41, 2, 9, 17, 25, 36]
    full = R.forward(CFG, w, toks)
    for n in (1, 4, 9):
        assert np.allclose(R.forward(CFG, w, toks[:n]), full[:n], atol=1e-10)
    for name in w:
        moved = dict(w, **{name: w[name][::-1] if len(w[name]) > 1 else -w[name]})
        if name.endswith("router.b"):
            moved[name] = w[name][::-1] * 30
        diff = np.abs(R.forward(CFG, moved, toks) - full).max()
        assert diff > 1e-4, name


def test_oracle_frequencies():
    """each branch of both scalings is taken, and its ends are where the
    definitions put them"""
    f = R.inverse_frequencies(16, 100.0)
    assert f[0] == 1.0 and np.isclose(f[4], 0.1)
    g = R.llama3_frequencies(f, **NM.LLAMA3) / f
    wave = 2 * np.pi / f
    assert (g[wave < 16] == 1).all() and np.allclose(g[wave > 64], 0.25)
    between = g[(wave >= 16) & (wave <= 64)]
    assert len(between) and ((between > 0.25) & (between < 1)).all()
    y, mult = R.yarn_frequencies(f, 16, 100.0, **NM.YARN)
    y = y / f
    assert y[0] == 1.0 and np.isclose(y[-1], 0.25) and (np.diff(y) <= 0).all()
    assert ((y > 0.25 + 1e-9) & (y < 1)).sum() >= 2 and np.isclose(mult, 0.1 * np.log(4.0) + 1.0)


def test_oracle_turned_values_see_distances_only():
    """With values turned by their positions and turned back by the query's, an
    output depends on distances: the same keys and values further on give it."""
    rng = np.random.default_rng(0)
    v = rng.standard_normal((6, 1, 10))
    f = R.inverse_frequencies(10, 50.0)
    out = []
    for start in (0, 40):
        pos = start + np.arange(6.0)
        out.append(R.turn_back(R.rotate(v, pos[:, None] * f, "half").sum(0)[None], pos[5:], 50.0, "half"))
    assert np.allclose(out[0], out[1])


def test_oracle_sink_takes_its_share():
    s = np.zeros((1, 3, 3))
    p = R.softmax_with_sink(s, R.visible(3, 0), np.array([np.log(2.0)]))
    assert np.allclose(p[0], [[1 / 3, 0, 0], [1 / 4, 1 / 4, 0], [1 / 5, 1 / 5, 1 / 5]])
    assert np.allclose(R.softmax_with_sink(s, R.visible(3, 2), None)[0, 2], [0, 0.5, 0.5])


def test_oracle_routing():
    """the chosen experts' weights are a softmax over them alone"""
    w = {"m.router": np.eye(4), "m.router.b": np.array([0.0, 0.0, 0.0, 5.0])}
    idx, wt = R.route(w, "m", np.array([[2.0, 3.0, 1.0, -3.0]]), 2)
    assert idx.tolist() == [[1, 0]] and np.allclose(wt, [[1 / (1 + np.exp(-1)), 1 / (1 + np.exp(1))]])
    assert R.route(w, "m", np.zeros((1, 4)), 1)[0].tolist() == [[3]]
