"""Vapipel configurations and checkpoints: what the reader takes and refuses
(no GPU: a valid configuration ends at the missing device)."""
import copy

import pytest

import flexflow_amd as fa
import flexflow_amd.ffmi as F
import vapipel_models as VM

CFG = VM.model_config(61, 48, 80, [VM.layer(3, 16, 8, 24, 0.3, 40),
                                   VM.layer(2, 8, 16, 24, 0.2, None, kv_from=0)])
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
    import ctypes
    n = ctypes.c_int(0)
    from hip_util import hip
    return hip().hipGetDeviceCount(ctypes.byref(n)) != 0 or n.value == 0


@pytest.mark.skipif(not no_gpu(), reason="the missing device is the expected end")
def test_valid_configurations_reach_the_device_check():
    assert NO_GPU in refusal(CFG)
    assert NO_GPU in refusal(CFG, full_precision=True)
    # kv_from naming the layer itself, and null, mean an own latent
    assert NO_GPU in refusal(edited(lambda c: c["layers"][1]["mixer"].update(kv_from=1)))
    assert NO_GPU in refusal(edited(lambda c: c["layers"][1]["mixer"].update(kv_from=None)))


@pytest.mark.parametrize("edit,what", [
    (lambda c: c.update(architecture="Nobody"), "Nobody"),
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c.pop("norm"), "norm.eps"),
    (lambda c: c.update(layers=[]), "layers"),
    (lambda c: c["layers"][0].update(type="convolution"), "convolution"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "layers[0].mixer"),
    (lambda c: c["layers"][1]["mixer"].update(kv_from=2), "layers[1].mixer.kv_from"),
    (lambda c: c["layers"][1]["mixer"].update(kv_rank=16), "layers[1].mixer.kv_from"),
    (lambda c: c["layers"][0]["mlp"].update(kind="gated"), "layers[0].mlp"),
    (lambda c: c["layers"][0]["mlp"].update(ff=12.5), "layers[0].mlp"),
])
def test_refused_configurations_name_the_place(edit, what):
    assert what in refusal(edited(edit))


def test_a_chain_of_shared_latents_is_refused():
    c = edited(lambda c: c["layers"].append(VM.layer(1, 8, 8, 24, 0.1, None, kv_from=1)))
    assert "layers[2].mixer.kv_from" in refusal(c)


def test_tree_and_beam_modes_are_not_offered():
    assert "unsupported" in refusal(CFG, mode="tree")


def test_load_config(tmp_path):
    VM.write_checkpoint(tmp_path, CFG, VM.random_weights(CFG, 1))
    assert fa.load_config(str(tmp_path)) == CFG


def test_oracle_decodes_as_it_prefills():
    """The plain implementation itself: a longer sequence leaves the earlier
    positions' logits alone, and every mechanism moves them."""
    import numpy as np
    import vapipel_ref as R
    w = VM.random_weights(CFG, 2, sharp=3.0)
    toks = [7, 3, 60, 0, 11, 11, 4]
    full = R.forward(CFG, w, toks)
    for n in (1, 4):
        assert np.allclose(R.forward(CFG, w, toks[:n]), full[:n], atol=1e-10)
    for name in ("pos", "l0.mix.g", "l0.mix.dkv.norm", "l1.mix.uk", "l1.norm1", "l0.mlp.up"):
        moved = dict(w, **{name: w[name][::-1]})
        assert np.abs(R.forward(CFG, moved, toks) - full).max() > 1e-3, name
