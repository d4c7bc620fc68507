"""Fesenex's gated product alone against an fp64 restatement, in every GEMM form
that its sizes reach (few rows, row blocks with and without a split of K, tiles)."""
import numpy as np
import pytest

import flexflow_amd.ffmi as F
from hip_util import Buf
from vapipel_models import bf16, bf16_bits

pytestmark = pytest.mark.gpu


@pytest.mark.parametrize("T,N,K", [(1, 32, 32), (7, 96, 64), (16, 1056, 320), (17, 544, 4096), (40, 2048, 96),
                                   (64, 160, 2080), (65, 416, 352), (100, 64, 8192), (168, 1024, 2048),
                                   (300, 96, 4128), (520, 2560, 512), (1024, 5120, 256), (700, 1024, 8192)])
@pytest.mark.parametrize("limit", [0.4, 7.0])
def test_linear_bf16_glu(T, N, K, limit):
    rng = np.random.default_rng(T + N + K)
    X, W = bf16(rng.uniform(-1, 1, (T, K))), bf16(rng.uniform(-1, 1, (2 * N, K)) * (6.0 / K ** 0.5))
    ref = X.astype(np.float64) @ W.astype(np.float64).T
    g, u = np.minimum(ref[:, :N], limit), np.clip(ref[:, N:], -limit, limit)
    want = g / (1.0 + np.exp(-1.702 * g)) * (u + 1.0)
    y = Buf.empty((T, N), np.uint16)
    print("glu", T, N, K, limit, flush=True)
    assert F.lib().ffmi_linear_bf16_glu(Buf(bf16_bits(X)).ptr, Buf(bf16_bits(W)).ptr, y.ptr, T, N, K, limit,
                                        None) == 0
    got = (y.get().astype(np.uint32) << 16).view(np.float32).astype(np.float64)
    # one rounding to bf16, and the sums' own error through the unit's slope
    slope = 2e-5 * (1.0 + np.abs(u) + np.abs(g))
    assert (np.abs(got - want) <= 2.0 ** -8 * np.abs(want) + slope).all(), np.abs(got - want).max()
