// gemm_bf16_plain.hip -- GEMM, bf16 in, bf16 out (kernels: gemm_kernels.h).
#include "gemm_kernels.h"

namespace ffmi {

hipError_t launch_gemm_bf16_plain(const uint16_t *X, const uint16_t *Wp, uint16_t *Y, float *ws,
                               size_t ws_bytes, int T, int N, int K, int flags, hipStream_t s,
                               Partials *defer) {
  return launch_gemm_kind<2>(X, Wp, Y, ws, ws_bytes, T, N, K, flags, s, defer, 0, nullptr);
}

}  // namespace ffmi
