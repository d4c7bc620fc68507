"""Nomutar's gated product alone against an fp64 restatement, in every GEMM form
that its sizes reach (few rows, row blocks with and without a split of K, tiles)."""
import numpy as np
import pytest

import flexflow_amd.ffmi as F
from hip_util import Buf
from vapipel_models import bf16, bf16_bits

pytestmark = pytest.mark.gpu


@pytest.mark.parametrize("T,N,K", [(1, 32, 32), (9, 96, 64), (16, 1120, 352), (18, 480, 4096), (39, 2048, 96),
                                   (64, 224, 2080), (67, 416, 384), (110, 64, 8192), (160, 1024, 2048),
                                   (310, 96, 4128), (515, 2560, 512), (1024, 5120, 288), (690, 1024, 8192)])
def test_linear_bf16_swiglu(T, N, K):
    rng = np.random.default_rng(T + N + K)
    X, W = bf16(rng.uniform(-1, 1, (T, K))), bf16(rng.uniform(-1, 1, (2 * N, K)) * (6.0 / K ** 0.5))
    ref = X.astype(np.float64) @ W.astype(np.float64).T
    g, u = ref[:, :N], ref[:, N:]
    want = g / (1.0 + np.exp(-g)) * u
    y = Buf.empty((T, N), np.uint16)
    print("swiglu", T, N, K, flush=True)
    assert F.lib().ffmi_linear_bf16_swiglu(Buf(bf16_bits(X)).ptr, Buf(bf16_bits(W)).ptr, y.ptr, T, N, K, None) == 0
    got = (y.get().astype(np.uint32) << 16).view(np.float32).astype(np.float64)
    # one rounding to bf16, and the sums' own error through the product's slope
    slope = 2e-5 * (1.0 + np.abs(u) + np.abs(g))
    assert (np.abs(got - want) <= 2.0 ** -8 * np.abs(want) + slope).all(), np.abs(got - want).max()
