// gemm_bf16_swiglu.hip -- GEMM, bf16 in, SiLU gate of paired gate / up tiles, bf16
// out (kernels: gemm_kernels.h).
#include "gemm_kernels.h"

namespace ffmi {

size_t gemm_bf16_swiglu_workspace_bytes(int T, int N, int K) { return gemm_slab_bytes(T, N, K, 1); }

hipError_t launch_gemm_bf16_swiglu(const uint16_t *X, const uint16_t *Wp, uint16_t *Y, float *ws,
                                   size_t ws_bytes, int T, int N, int K, int flags, int y_width,
                                   hipStream_t s) {
  FuseArgs f;
  f.y_width = y_width;
  return launch_gemm_kind<6>(X, Wp, Y, ws, ws_bytes, T, N, K, flags, s, nullptr, 0, &f);
}

}  // namespace ffmi
