// memory_util.h -- what both forms of the matrix memories share (memory.h).
#pragma once
#include "device_util.h"
#include "memory.h"

namespace ffmi {

__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
// columns of q | k | v
__device__ __forceinline__ int memory_columns(const Memory &a) { return 2 * a.G * a.dg + a.H * a.vg; }
// log of the decay of channel c < dg of head h from its logit (bias not in yet)
template <MemoryRule RULE>
__device__ __forceinline__ float log_decay(const Memory &a, int h, int c, float z) {
  if (c >= a.dim) return 0.f;
  z += a.dbias[(size_t)h * a.dg + c];
  if constexpr (RULE == kMemoryDelta) return -a.rate[h] * softplus_f(z);
  else return -a.inv_tau * softplus_f(-z);
}
// a head's log input and forget gates of one token
__device__ __forceinline__ void memory_gates(const Memory &a, int t, int h, float &i, float &f) {
  const size_t slab = (size_t)a.T * a.y.NP, row = (size_t)t * a.y.NP;
  i = a.cap * tanhf(__fdiv_rn(sum_at(a.y, slab, row + a.col_i + h) + a.bi[h], a.cap));
  f = a.cap * tanhf(__fdiv_rn(sum_at(a.y, slab, row + a.col_f + h) + a.bf[h], a.cap));
  f = -softplus_f(-f);
}

}  // namespace ffmi
