// gemm_bf16_glu.hip -- GEMM, bf16 in, clamped gated unit of paired gate / up
// tiles, bf16 out (kernels: gemm_kernels.h).
#include "gemm_kernels.h"

namespace ffmi {

size_t gemm_bf16_glu_workspace_bytes(int T, int N, int K) { return gemm_slab_bytes(T, N, K, 1); }

hipError_t launch_gemm_bf16_glu(const uint16_t *X, const uint16_t *Wp, uint16_t *Y, float *ws,
                                size_t ws_bytes, int T, int N, int K, int flags, float limit,
                                hipStream_t s) {
  FuseArgs f;
  f.limit = limit;
  return launch_gemm_kind<5>(X, Wp, Y, ws, ws_bytes, T, N, K, flags, s, nullptr, 0, &f);
}

}  // namespace ffmi
