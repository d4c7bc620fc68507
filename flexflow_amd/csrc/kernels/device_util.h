// device_util.h -- small device functions of the bf16 / fp32 model kernels.
#pragma once
#include "../ffmi_internal.h"

namespace ffmi {

__device__ __forceinline__ uint4 pack8_bf16(const f4 &a, const f4 &b) {
  uint4 o;
  o.x = f2bf(a[0]) | ((uint32_t)f2bf(a[1]) << 16);
  o.y = f2bf(a[2]) | ((uint32_t)f2bf(a[3]) << 16);
  o.z = f2bf(b[0]) | ((uint32_t)f2bf(b[1]) << 16);
  o.w = f2bf(b[2]) | ((uint32_t)f2bf(b[3]) << 16);
  return o;
}
__device__ __forceinline__ void unpack8_bf16(const uint4 &v, f4 &a, f4 &b) {
  const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float lo = __builtin_bit_cast(float, w[i] << 16);
    const float hi = __builtin_bit_cast(float, w[i] & 0xffff0000u);
    if (i < 2) a[2 * i] = lo, a[2 * i + 1] = hi;
    else b[2 * i - 4] = lo, b[2 * i - 3] = hi;
  }
}


__device__ __forceinline__ float ld_elem(const uint16_t *p) { return bf2f(*p); }
__device__ __forceinline__ float ld_elem(const float *p) { return *p; }
__device__ __forceinline__ void st_elem(uint16_t *p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void st_elem(float *p, float v) { *p = v; }

__device__ __forceinline__ float sigmoid_f(float v) { return __fdiv_rn(1.0f, 1.0f + expf(-v)); }
__device__ __forceinline__ float silu_f(float v) { return v * sigmoid_f(v); }
// value and remainder in bf16
__device__ __forceinline__ void split2(float v, __bf16 &hi, __bf16 &lo) {
  hi = (__bf16)v;
  lo = (__bf16)(v - (float)hi);
}
// element `at` of deferred sums
__device__ __forceinline__ float sum_at(const Partials &y, size_t slab, size_t at) {
  float v = y.p[at];
  for (int s = 1; s < y.S; ++s) v += y.p[at + s * slab];
  return v;
}

template <int NT>
__device__ __forceinline__ float row_sum(float v, float *sh) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
  if ((threadIdx.x & 63) == 0) sh[threadIdx.x >> 6] = v;
  __syncthreads();
  v = sh[0];
#pragma unroll
  for (int i = 1; i < NT / 64; ++i) v += sh[i];
  return v;
}
__device__ __forceinline__ float inv_rms(float ss, int n, float eps) {
  return __fdiv_rn(1.0f, sqrtf(__fdiv_rn(ss, (float)n) + eps));
}

// cosine and sine of so many turns
__device__ __forceinline__ void turn_by(double turns, float &c, float &s) {
  sincospif(2.0f * (float)(turns - rint(turns)), &s, &c);
}

}  // namespace ffmi
