"""Pekarax configurations and checkpoints: what the reader takes and refuses (no
GPU: a valid configuration ends at the missing device), and the plain
implementation itself."""
import copy
import ctypes

import numpy as np
import pytest

import flexflow_amd as fa
import flexflow_amd.ffmi as F
import pekarax_models as PM
import pekarax_ref as R

CFG = PM.model_config(61, 48, [
    PM.experts(PM.delta(4, 2, 16, 8, conv=3), 6, 2, 24, identity=2, groups=(4, 2)),
    PM.experts(PM.parallel((2, 1, 16, 12, 0.9, 8, 50.0, 2), (2, 8, 12, 4.0)), 5, 2, 24),
    PM.gla(2, 12, 8)])
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


def router(c, i=0):
    return c["layers"][i]["mlp"]["router"]


@pytest.mark.skipif(not no_gpu(), reason="the missing device is the expected end")
@pytest.mark.parametrize("edit", [
    lambda c: None,
    lambda c: c["layers"].reverse(),
    lambda c: c.update(layers=c["layers"][2:]),
    lambda c: c["layers"][0].update(mlp=None),
    lambda c: c["layers"][2].pop("mlp"),
    lambda c: router(c).pop("groups"),
    lambda c: router(c).update(groups=None),
    lambda c: router(c).update(top=4),
    lambda c: router(c, 1).update(top=5),
    lambda c: router(c).update(identity=0, groups=dict(count=3, keep=1)),
    lambda c: router(c, 1).pop("identity"),
    lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=0),
    lambda c: c["layers"][1]["mixer"]["left"].update(conv=1),
    lambda c: c["layers"][0]["mixer"].update(conv=1, kv_heads=4),
])
def test_valid_configurations_reach_the_device_check(edit):
    assert NO_GPU in refusal(edited(edit))
    assert NO_GPU in refusal(edited(edit), full_precision=True)


@pytest.mark.parametrize("edit,what", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c.pop("norm"), "norm.eps"),
    (lambda c: c.pop("postln_alpha"), "postln_alpha"),
    (lambda c: c.update(layers=[]), "layers"),
    (lambda c: c["layers"][0].update(type="delta"), "layers[0].type 'delta'"),
    (lambda c: c["layers"][0].pop("mixer"), "layers[0].mixer"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "layers[0].mixer"),
    (lambda c: c["layers"][0]["mixer"].update(conv=0), "layers[0].mixer.conv"),
    (lambda c: c["layers"][0]["mixer"].update(dim=0), "layers[0].mixer"),
    (lambda c: c["layers"][1]["mixer"].pop("left_scale"), "layers[1].mixer"),
    (lambda c: c["layers"][1]["mixer"].pop("left"), "layers[1].mixer.left"),
    (lambda c: c["layers"][1]["mixer"]["left"].pop("scale"), "layers[1].mixer.left"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(heads=3, kv_heads=2), "layers[1].mixer.left"),
    (lambda c: c["layers"][1]["mixer"]["left"].pop("conv"), "layers[1].mixer.left.conv"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=18), "layers[1].mixer.left.rot"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7), "layers[1].mixer.left.rot"),
    (lambda c: c["layers"][1]["mixer"]["left"].pop("rot"), "layers[1].mixer.left.rot"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(gate_cap=0.0), "layers[1].mixer.right"),
    (lambda c: c["layers"][1]["mixer"]["right"].pop("vdim"), "layers[1].mixer.right"),
    (lambda c: c["layers"][2]["mixer"].update(tau=-1.0), "layers[2].mixer"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "layers[0].mlp.kind 'dense'"),
    (lambda c: c["layers"][0]["mlp"].pop("expert"), "layers[0].mlp.expert"),
    (lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"), "layers[0].mlp.expert"),
    (lambda c: router(c).update(experts=0), "layers[0].mlp.router"),
    (lambda c: router(c).update(top=5), "layers[0].mlp.router"),
    (lambda c: router(c).update(identity=-1), "layers[0].mlp.router.identity"),
    (lambda c: router(c)["groups"].update(count=3), "layers[0].mlp.router.groups"),
    (lambda c: router(c)["groups"].update(keep=5), "layers[0].mlp.router.groups"),
    (lambda c: router(c)["groups"].pop("keep"), "layers[0].mlp.router.groups"),
])
def test_refused_configurations_name_the_place(edit, what):
    assert what in refusal(edited(edit))


def test_tree_and_beam_modes_are_not_offered():
    assert "unsupported" in refusal(CFG, mode="tree")


def test_load_config(tmp_path):
    PM.write_checkpoint(tmp_path, CFG, PM.random_weights(CFG, 1))
    assert fa.load_config(str(tmp_path)) == CFG


# ---- the plain implementation ----
def test_oracle_decodes_as_it_prefills():
    """A longer sequence leaves the earlier positions' logits alone, and every
    tensor that a sequence of this length reaches moves them."""
    w = PM.random_weights(CFG, 2)
    toks = [7, 3, 60, 0, 11, 11, 4, 33, 20, 58, 41, 2, 9, 17, 25, 36]
    full = R.forward(CFG, w, toks)
    for n in (1, 4, 9):
        assert np.allclose(R.forward(CFG, w, toks[:n]), full[:n], atol=1e-10)
    taken = set()
    for i in (0, 1):
        p = "l%d.mlp." % i
        x, layers = w["embed"][np.asarray(toks)], []
        R.forward(CFG, w, toks, layers)
        for row in (layers[i] if i else layers[0]):
            taken |= {p + "e%d." % e for e in R.route(w[p + "router"] @ row, w[p + "correction"], router(CFG, i))[0]}
    for name in w:
        if ".mlp.e" in name and name[:name.rindex(".") + 1] not in taken:
            continue
        moved = dict(w, **{name: w[name][::-1] if len(w[name]) > 1 else -w[name]})
        if name.endswith("correction"):
            moved[name] = np.linspace(-9.0, 9.0, len(w[name]))
        diff = np.abs(R.forward(CFG, moved, toks) - full).max()
        assert diff > 1e-4, name


def test_oracle_rotation_keeps_relative_positions():
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((2, 1, 1, 10))
    x = R.rotate(np.repeat(q, 30, 0), 8, 50.0), R.rotate(np.repeat(k, 30, 0), 8, 50.0)
    dots = [(x[0][i + 5] * x[1][i]).sum() for i in (0, 7, 20)]
    assert np.allclose(dots, dots[0]) and np.allclose(x[0][:, :, 8:], q[:, :, 8:])


def test_oracle_delta_rule_recalls_what_it_wrote():
    """With unit step and no decay, reading a key gives its last value, whatever was
    written under it before."""
    k = np.eye(3)[[0, 1, 0, 2]]
    v = np.arange(8.0).reshape(4, 2)
    out = R.delta_read(np.eye(3)[[0, 0, 0, 0]], k, v, np.ones(4), np.ones((4, 3)))
    assert np.allclose(out, [v[0], v[0], v[2], v[2]])


def test_oracle_normalised_memory_is_a_weighted_mean():
    """Equal keys: the output is the values' mean, weighted by gates, wherever that
    exceeds the least denominator; the running maximum changes nothing."""
    k = np.ones((4, 1))
    i, f, v = np.array([3.0, 1.0, 9.0, 2.0]), np.log([0.9, 0.5, 0.8, 0.7]), np.arange(4.0)[:, None]
    out = R.mlstm_read(k, k, v, i, f)
    F = np.cumsum(f)
    for t in range(4):
        wt = np.exp(F[t] - F[:t + 1] + i[:t + 1])
        assert np.allclose(out[t], (wt @ v[:t + 1]) / wt.sum(), rtol=1e-4, atol=1e-6)
    small = R.mlstm_read(k, k, v + 1.0, i - 20.0, f)
    assert np.allclose(small[0], np.exp(-17.0) * 1.0, rtol=1e-5)


def test_oracle_gated_memory_forgets_by_channel():
    q, k = np.ones((3, 2)), np.eye(2)[[0, 1, 1]]
    out = R.gla_read(q, k, np.array([[1.0], [10.0], [0.0]]), np.array([[0.5, 1.0]] * 3))
    assert np.allclose(out[:, 0], [1.0, 10.5, 10.25])


def test_oracle_routing():
    r = dict(experts=4, identity=2, top=2, scale=2.0, groups=dict(count=3, keep=1))
    z, c = np.log([4.0, 1.0, 2.0, 2.0, 3.0, 1.0]), np.array([-1.0, 0, 0, 0, -1.0, 0])
    picked, wt = R.route(z, c, r)  # groups by their best corrected score: 1/13, 2/13, 1/13
    assert picked == [2, 3] and np.allclose(wt, [1.0, 1.0])
    picked, wt = R.route(z, 0 * c, dict(r, groups=None))
    assert picked == [0, 4] and np.allclose(wt, [8 / 7, 6 / 7])
    # corrected scores below zero still beat what is left out
    picked, _ = R.route(z, np.full(6, -5.0), r)
    assert picked == [0, 1]
