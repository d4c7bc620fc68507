"""Fesenex configurations and checkpoints: what the reader takes and refuses
(no GPU: a valid configuration ends at the missing device), and the plain
implementation itself."""
import copy
import ctypes

import numpy as np
import pytest

import fesenex_models as FM
import fesenex_ref as R
import flexflow_amd as fa
import flexflow_amd.ffmi as F

MODEL = FM.model_config(61, 48, [FM.attention(4, 2, 16, 8, 0.3, q_temp=(0.5, 3), v_mix=True, ff=40),
                                 FM.lightning(2, 8, 16, [0.5, 0.9]),
                                 FM.attention(2, 2, 12, 8, 0.2, bias_max=5, v_mix=True, rel_rows=4)])
CFG = MODEL[0]
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
def test_valid_configurations_reach_the_device_check():
    assert NO_GPU in refusal(CFG)
    assert NO_GPU in refusal(CFG, full_precision=True)
    # no temperature, absent or null; no mixing; layers of one kind only
    assert NO_GPU in refusal(edited(lambda c: c["layers"][0]["mixer"].pop("q_temp")))
    assert NO_GPU in refusal(edited(lambda c: c["layers"][0]["mixer"].update(q_temp=None)))
    assert NO_GPU in refusal(edited(lambda c: c["layers"][0]["mixer"].pop("v_mix")))
    assert NO_GPU in refusal(edited(lambda c: c.update(layers=c["layers"][1:2])))
    assert NO_GPU in refusal(edited(lambda c: c.update(layers=c["layers"][:1])))


@pytest.mark.parametrize("edit,what", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c.pop("norm"), "norm.eps"),
    (lambda c: c.update(embedding=dict()), "embedding.scale"),
    (lambda c: c.update(layers=[]), "layers"),
    (lambda c: c["layers"][0].update(type="convolution"), "convolution"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "layers[0].mixer"),
    (lambda c: c["layers"][0]["mixer"].pop("bias_max"), "layers[0].mixer"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "layers[0].mixer"),
    (lambda c: c["layers"][0]["mixer"].update(q_temp=dict(coef=1.0)), "layers[0].mixer.q_temp"),
    (lambda c: c["layers"][0]["mixer"].update(v_mix=1), "layers[0].mixer.v_mix"),
    (lambda c: c["layers"][2]["mixer"].update(vdim=16), "layers[2].mixer.v_mix"),
    (lambda c: c["layers"][1]["mixer"].update(decay=[0.5]), "layers[1].mixer.decay"),
    (lambda c: c["layers"][0]["mlp"].update(kind="experts"), "layers[0].mlp"),
    (lambda c: c["layers"][0]["mlp"].pop("limit"), "layers[0].mlp"),
])
def test_refused_configurations_name_the_place(edit, what):
    assert what in refusal(edited(edit))


def test_tree_and_beam_modes_are_not_offered():
    assert "unsupported" in refusal(CFG, mode="tree")


def test_load_config(tmp_path):
    FM.write_checkpoint(tmp_path, CFG, FM.random_weights(MODEL, 1))
    assert fa.load_config(str(tmp_path)) == CFG


def test_oracle_decodes_as_it_prefills():
    """A longer sequence leaves the earlier positions' logits alone, and every
    tensor moves them."""
    w = FM.random_weights(MODEL, 2, sharp=3.0)
    toks = [7, 3, 60, 0, 11, 11, 4]
    full = R.forward(CFG, w, toks)
    for n in (1, 4):
        assert np.allclose(R.forward(CFG, w, toks[:n]), full[:n], atol=1e-10)
    unused = {"l0.mix.vmix"}  # the first mixing layer has nothing to mix
    for name in w:
        moved = dict(w, **{name: w[name][::-1] if w[name].ndim else w[name] * 0.5})
        diff = np.abs(R.forward(CFG, moved, toks) - full).max()
        assert (diff == 0) if name in unused else diff > 1e-3, name


def test_oracle_linear_attention_is_a_weighted_sum():
    """The recurrence against its closed form."""
    rng = np.random.default_rng(0)
    q, k, v = rng.standard_normal((9, 2, 5)), rng.standard_normal((9, 2, 5)), rng.standard_normal((9, 2, 3))
    d = np.array([0.7, 1.0])
    o = R.lightning_states(q, k, v, d)
    for h in range(2):
        for i in range(9):
            want = sum(d[h] ** (i - j) * (q[i, h] @ k[j, h]) * v[j, h] for j in range(i + 1))
            assert np.allclose(o[i, h], want)
