// memory_util.h -- what both forms of the matrix memories share (memory.h).
#pragma once
#include "device_util.h"
#include "memory.h"

namespace ffmi {

__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
// columns of q | k | v
__device__ __forceinline__ int memory_columns(const Memory &a) { return 2 * a.G * a.dg + a.H * a.vg; }
// a decay from its logit, in full precision (rate: of the head)
template <MemoryRule RULE>
__device__ __forceinline__ float decay_of(const Memory &a, float rate, float z) {
  if constexpr (RULE == kMemoryDelta) return expf(-rate * softplus_f(z));
  else return expf(-a.inv_tau * softplus_f(-z));
}
// bf16 model: its log, base 2, by the base-2 instructions; what the logarithm loses of
// small values (6e-8) is what a decay next to 1 has no bits for
constexpr float kLog2e = 1.4426950408889634f;
__device__ __forceinline__ float ex2(float v) { return __builtin_amdgcn_exp2f(v); }
__device__ __forceinline__ float softplus2(float z) {
  z *= kLog2e;
  return fmaxf(z, 0.f) + __builtin_amdgcn_logf(1.f + ex2(-fabsf(z)));
}
template <MemoryRule RULE>
__device__ __forceinline__ float log2_decay(const Memory &a, float rate, float z) {
  if constexpr (RULE == kMemoryDelta) return -rate * softplus2(z);
  else return -a.inv_tau * softplus2(-z);
}
// a head's log input and forget gates of one token
__device__ __forceinline__ void memory_gates(const Memory &a, int t, int h, float &i, float &f) {
  const size_t slab = (size_t)a.T * a.y.NP, row = (size_t)t * a.y.NP;
  i = a.cap * tanhf(__fdiv_rn(sum_at(a.y, slab, row + a.col_i + h) + a.bi[h], a.cap));
  f = a.cap * tanhf(__fdiv_rn(sum_at(a.y, slab, row + a.col_f + h) + a.bf[h], a.cap));
  f = -softplus_f(-f);
}

}  // namespace ffmi
