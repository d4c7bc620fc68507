// gemm_bf16_f32.hip -- GEMM, bf16 in, fp32 slabs out (kernels: gemm_kernels.h).
#include "gemm_kernels.h"

namespace ffmi {

size_t gemm_bf16_workspace_bytes(int T, int N, int K) {
  return std::max(gemm_slab_bytes(T, N, K, 0), (size_t)T * ((N + 15) / 16) * 16 * sizeof(float));
}

hipError_t launch_gemm_bf16_f32(const uint16_t *X, const uint16_t *Wp, uint16_t *Y, float *ws,
                               size_t ws_bytes, int T, int N, int K, int flags, hipStream_t s,
                               Partials *defer) {
  return launch_gemm_kind<4>(X, Wp, Y, ws, ws_bytes, T, N, K, flags, s, defer, 0, nullptr);
}

}  // namespace ffmi
