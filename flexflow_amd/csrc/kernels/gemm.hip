// gemm.hip -- the fp16 GEMM entry points (kernels: gemm_kernels.h).
#include "gemm_kernels.h"

namespace ffmi {

size_t gemm_workspace_bytes(int T, int N, int K, int epilogue) {
  return gemm_slab_bytes(T, N, K, epilogue & ~(FFMI_X_PACKED | FFMI_Y_PACKED | FFMI_W_STREAM));
}

hipError_t launch_partials_reduce(const Partials &p, uint16_t *Y, int T, int N, hipStream_t s) {
  if (T <= 0 || p.S <= 0) return hipSuccess;
  // (> 8: the per-head o-projection slabs of a small model, OprojArgs)
  if (p.S > 16 || p.NP % 16 || N > p.NP) return hipErrorInvalidValue;
  const long total = (long)T * ((N + 3) / 4);
  const unsigned blocks = (unsigned)((total + 255) / 256);
#define FFMI_PRED(MS)                                                                          \
  hipLaunchKernelGGL((gemm_reduce_kernel<0, MS>), dim3(blocks), dim3(256), 0, s, p.p, Y, T, N, \
                     p.NP / 16, p.S, 0, 0.f)
  if (p.S <= 2) FFMI_PRED(2);
  else if (p.S <= 4) FFMI_PRED(4);
  else if (p.S <= 8) FFMI_PRED(8);
  else FFMI_PRED(16);
#undef FFMI_PRED
  return hipGetLastError();
}

hipError_t launch_gemm(const uint16_t *X, const uint16_t *Wp, uint16_t *Y, float *ws,
                       size_t ws_bytes, int T, int N, int K, int epilogue, hipStream_t s,
                       Partials *defer, int wpitch, const FuseArgs *fuse) {
  if ((epilogue & ~(FFMI_X_PACKED | FFMI_Y_PACKED | FFMI_W_STREAM)) == FFMI_EPI_SILU_MUL)
    return launch_gemm_kind<1>(X, Wp, Y, ws, ws_bytes, T, N, K, epilogue, s, defer, wpitch, fuse);
  return launch_gemm_kind<0>(X, Wp, Y, ws, ws_bytes, T, N, K, epilogue, s, defer, wpitch, fuse);
}

// Packed activation tiles: Xp[mt][kt][lane][8] = X[mt*16 + (lane&15)][kt*32 + 8(lane>>4) + e]
// (rows >= T zero) -- the MFMA operand fragment order of the weights (weights.hip),
// so a GEMM reads each activation fragment as one contiguous 1 KiB.
__global__ void pack_act_kernel(const uint16_t *__restrict__ X, uint16_t *__restrict__ Xp, int T,
                                int K, int KT) {
  const int mt = blockIdx.y, kt = blockIdx.x, l = threadIdx.x;
  const int r = mt * 16 + (l & 15);
  uint4 v = make_uint4(0, 0, 0, 0);
  if (r < T) v = *reinterpret_cast<const uint4 *>(X + (size_t)r * K + kt * 32 + 8 * (l >> 4));
  *reinterpret_cast<uint4 *>(Xp + (((size_t)mt * KT + kt) * 64 + l) * 8) = v;
}

size_t packed_act_bytes(int T, int K) { return (size_t)((T + 15) / 16) * 16 * K * 2; }

hipError_t launch_pack_act(const uint16_t *X, uint16_t *Xp, int T, int K, hipStream_t s) {
  if (T <= 0) return hipSuccess;
  hipLaunchKernelGGL(pack_act_kernel, dim3(K / 32, (T + 15) / 16), dim3(64), 0, s, X, Xp, T, K,
                     K / 32);
  return hipGetLastError();
}

// diagnostics: stamps of the last FFMI_GEMM_STAMP launch (8 int64 per wave)
long gemm_debug_stamps(long long *dst, long max_waves) {
  long long *buf = stamp_buf();
  const long n = g_stamp_entries < max_waves ? g_stamp_entries : max_waves;
  if (!buf || n <= 0) return 0;
  if (hipDeviceSynchronize() != hipSuccess) return -1;
  if (hipMemcpy(dst, buf, (size_t)n * 8 * sizeof(long long), hipMemcpyDeviceToHost) != hipSuccess)
    return -1;
  return n;
}

}  // namespace ffmi
