// packing.hip -- checkpoint matrices and activations to the layouts the
// kernels take (packing.h).
#include "packing.h"

namespace ffmi {

// the index of destination element (n, k) in src; -1: padding
__device__ __forceinline__ long pack_index(int ld, const PackSpec &p, int n, int k) {
  const int hn = n / p.np, hk = k / p.kp;
  int jn = n % p.np, jk = k % p.kp;
  if (jn < p.row_pairs) jn = (jn >> 1) + (jn & 1) * (p.row_pairs >> 1);
  if (jk < p.col_pairs) jk = (jk >> 1) + (jk & 1) * (p.col_pairs >> 1);
  if (hn >= p.rows || jn >= p.nb || hk >= p.cols || jk >= p.kb) return -1;
  if (p.transpose) return ((long)(hn * p.cols + hk) * p.kb + jk) * ld + jn;
  return (long)(hn * p.nb + jn) * ld + hk * p.kb + jk;
}
__device__ __forceinline__ uint16_t pack_elem(const uint16_t *src, int ld, const PackSpec &p, int n,
                                              int k) {
  const long at = pack_index(ld, p, n, k);
  return at < 0 ? 0 : src[at];
}
__global__ void pack_bf16_kernel(const uint16_t *__restrict__ src, int ld, PackSpec p,
                                 uint16_t *__restrict__ dst, int NT, int KT, size_t ts, size_t ks) {
  const long gid = blockIdx.x * (long)blockDim.x + threadIdx.x;
  if (gid >= (long)NT * KT * 64) return;
  const int lane = (int)(gid & 63), kt = (int)((gid >> 6) % KT), nt = (int)((gid >> 6) / KT);
  const int n = nt * 16 + (lane & 15), k = kt * 32 + 8 * (lane >> 4);
  uint32_t v[4];
#pragma unroll
  for (int j = 0; j < 4; ++j)
    v[j] = pack_elem(src, ld, p, n, k + 2 * j) |
           ((uint32_t)pack_elem(src, ld, p, n, k + 2 * j + 1) << 16);
  *reinterpret_cast<uint4 *>(dst + nt * ts + kt * ks + lane * 8) = make_uint4(v[0], v[1], v[2], v[3]);
}
hipError_t launch_pack_bf16(const uint16_t *src, int ld, const PackSpec &p, uint16_t *dst,
                            int tile_offset, int pitch, bool perhead, hipStream_t s,
                            int tile_step) {
  const int N = p.rows * p.np, K = p.cols * p.kp;
  if (N % 16 || K % 32) return hipErrorInvalidValue;
  const int NT = N / 16, KT = K / 32;
  const size_t ts = perhead ? (size_t)KT * 512 : w_tile_stride(p.kt ? p.kt : KT);
  const size_t ks = perhead ? 512 : w_k_stride(pitch);
  dst += p.k0 * ks;
  hipLaunchKernelGGL(pack_bf16_kernel, dim3((unsigned)(((long)NT * KT * 64 + 255) / 256)),
                     dim3(256), 0, s, src, ld, p, dst + tile_offset * ts, NT, KT,
                     tile_step * ts, ks);
  return hipGetLastError();
}
__global__ void pack_f32_kernel(const uint16_t *__restrict__ src, int ld, PackSpec p,
                                float *__restrict__ dst, int N, int K, int ldd) {
  const long i = blockIdx.x * (long)blockDim.x + threadIdx.x;
  if (i >= (long)N * K) return;
  const long at = pack_index(ld, p, (int)(i / K), (int)(i % K));
  dst[i / K * ldd + i % K] = at < 0 ? 0.f : bf2f(src[at]) + p.plus;
}
hipError_t launch_pack_f32(const uint16_t *src, int ld, const PackSpec &p, float *dst,
                           hipStream_t s) {
  const int N = p.rows * p.np, K = p.cols * p.kp;
  hipLaunchKernelGGL(pack_f32_kernel, dim3((unsigned)(((long)N * K + 255) / 256)), dim3(256), 0, s,
                     src, ld, p, dst + p.k0 * 32, N, K, p.kt ? p.kt * 32 : K);
  return hipGetLastError();
}

__global__ void pack_act_bf16_kernel(const uint16_t *__restrict__ X, uint16_t *__restrict__ Xp,
                                     int T, int K) {
  const int kt = blockIdx.x, mt = blockIdx.y, l = threadIdx.x, r = mt * 16 + (l & 15);
  uint4 v = make_uint4(0, 0, 0, 0);
  if (r < T) v = *reinterpret_cast<const uint4 *>(X + (size_t)r * K + kt * 32 + 8 * (l >> 4));
  *reinterpret_cast<uint4 *>(Xp + act_packed_off(r, kt * 32 + 8 * (l >> 4), K)) = v;
}
hipError_t launch_pack_act_bf16(const uint16_t *X, uint16_t *Xp, int T, int K, hipStream_t s) {
  if (T <= 0 || K % 32) return hipErrorInvalidValue;
  hipLaunchKernelGGL(pack_act_bf16_kernel, dim3(K / 32, (T + 15) / 16), dim3(64), 0, s, X, Xp, T, K);
  return hipGetLastError();
}

}  // namespace ffmi
