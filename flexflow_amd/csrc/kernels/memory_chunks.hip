// memory_chunks.hip -- matrix memories in chunks of 64 tokens on MFMA (memory.h).
//
// With G_i the sum of the log decays of a chunk's tokens up to i (per key channel; normed:
// one for all) and S the state before the chunk:
//   p_ij = sum over channels of q_i k_j exp(G_i - G_j), j <= i
//   u    = v, or delta: u_i = beta_i (v_i - (k_i exp(G_i))^T S - sum over j < i of a_ij u_j)
//          with a_ij as p_ij with k_i for q_i; so u = T (beta v) - T (beta k exp(G)) S with
//          T = (1 + beta a)^-1, unit lower triangular
//   o_i  = (q_i exp(G_i))^T S + sum over j <= i of p_ij u_j
//   S'   = exp(G_last) S + sum over j of (k_j exp(G_last - G_j)) u_j^T
// Launches: delta: convolved rows; normed: gates; then what does not need S, all chunks
// side by side; then the pass over a span's chunks with the state in registers.
//
// No exponent is ever positive beyond kSpread: a chunk's four blocks of 16 tokens take their
// decays from the blocks' borders, and a block's own 16 x 16 products from its start while
// its decays add up to less than that, else one exponential per pair and channel.
// Logs of decays have base 2.
#include <algorithm>

#include "conv_rows.h"
#include "memory_util.h"

namespace ffmi {

namespace {

typedef short s4 __attribute__((ext_vector_type(4)));
constexpr int C = kMemoryChunk;
constexpr float kSpread = 80.f;  // base 2: far from fp32's and bf16's range on either side

__device__ __forceinline__ f4 mma(bf8 a, bf8 b, f4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }

// operand of 8 k-values from row-major LDS rows of LD: column c0 + (lane & 15), rows
// kb * 32 + 8g .. 8g + 7
template <int LD>
__device__ __forceinline__ bf8 read_columns(const uint16_t *tile, int kb, int c0) {
  const int lane = threadIdx.x & 63, g = lane >> 4, l15 = lane & 15;
  const uint16_t *p = tile + (kb * 32 + 8 * g + (l15 >> 2)) * LD + c0 + 4 * (l15 & 3);
  const s4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4 *)(p));
  const s4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4 *)(p + 4 * LD));
  return __builtin_bit_cast(bf8, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
}
__device__ __forceinline__ void sum8(const Partials &y, size_t slab, size_t at, f4 (&v)[2]) {
  v[0] = *reinterpret_cast<const f4 *>(y.p + at), v[1] = *reinterpret_cast<const f4 *>(y.p + at + 4);
  for (int s = 1; s < y.S; ++s) {
    v[0] += *reinterpret_cast<const f4 *>(y.p + at + s * slab);
    v[1] += *reinterpret_cast<const f4 *>(y.p + at + s * slab + 4);
  }
}
__device__ __forceinline__ uint2 pack4(const f4 &v) {
  return make_uint2(f2bf(v[0]) | ((uint32_t)f2bf(v[1]) << 16), f2bf(v[2]) | ((uint32_t)f2bf(v[3]) << 16));
}

__device__ __forceinline__ void load8(const float *p, f4 (&v)[2]) {
  v[0] = *reinterpret_cast<const f4 *>(p), v[1] = *reinterpret_cast<const f4 *>(p + 4);
}
// the span whose chunk `c` is (counted over the step's long spans); a wave looks for it
__device__ __forceinline__ int span_of_chunk(const PagedSpan *spans, int num, int c) {
  for (int b = 0; b < num; b += 64) {
    const int i = b + (threadIdx.x & 63);
    bool hit = false;
    if (i < num) {
      const PagedSpan sp = spans[i];
      hit = sp.n > kShortSpan && c >= sp.chunk0 && c < sp.chunk0 + (sp.n + C - 1) / C;
    }
    const uint64_t m = __ballot(hit);
    if (m) return __builtin_amdgcn_readfirstlane(b + __ffsll((unsigned long long)m) - 1);
  }
  return -1;
}

// normed: decay, key factor (logs, base 2) and m of every token of a long span; a workgroup
// per (head, span), m by a scan of the maps m -> max(m + f, i)
__global__ __launch_bounds__(256) void memory_gates_kernel(const char *__restrict__ blob, int off_spans, Memory a,
                                                           MemoryScratch w, int limit) {
  __shared__ float sa[2][256], sb[2][256];
  const PagedSpan sp = reinterpret_cast<const PagedSpan *>(blob + off_spans)[blockIdx.y];
  if (sp.n <= limit) return;
  const int tid = threadIdx.x, h = blockIdx.x, per = (sp.n + 255) / 256;
  const int b = min(tid * per, sp.n), e = min(b + per, sp.n), bank = sp.bank;
  float add = 0.f, top = -INFINITY;
  for (int t = b; t < e; ++t) {
    float i, f;
    memory_gates(a, sp.t0 + t, h, i, f);
    add += f, top = fmaxf(top + f, i);
  }
  int cur = 0;
  sa[0][tid] = add, sb[0][tid] = top;
  __syncthreads();
  for (int o = 1; o < 256; o <<= 1, cur ^= 1) {
    if (tid >= o) {
      const float pa = sa[cur][tid - o], pb = sb[cur][tid - o];
      top = fmaxf(pb + add, top), add += pa;
    }
    sa[cur ^ 1][tid] = add, sb[cur ^ 1][tid] = top;
    __syncthreads();
  }
  float m = sp.pos0 > 0 ? a.peak[((size_t)sp.slot * 2 + bank) * a.H + h] : 0.f;
  if (tid > 0) m = fmaxf(m + sa[cur][tid - 1], sb[cur][tid - 1]);
  for (int t = b; t < e; ++t) {
    float i, f;
    memory_gates(a, sp.t0 + t, h, i, f);
    const float mn = fmaxf(f + m, i);
    float *g = w.gates + ((size_t)(sp.t0 + t) * a.H + h) * 3;
    g[0] = (f + m - mn) * kLog2e, g[1] = (i - mn) * kLog2e, g[2] = mn;
    m = mn;
    if (t + 1 == sp.n) a.peak[((size_t)sp.slot * 2 + (bank ^ 1)) * a.H + h] = m;
  }
}

// A workgroup per (chunk, head); wave b has the chunk's block of 16 tokens b.
template <MemoryRule RULE, int KS>
__global__ __launch_bounds__(256, KS <= 4 ? 2 : 1) void memory_chunk_kernel(const char *__restrict__ blob, int off_spans,
                                                                            int num_spans, Memory a, MemoryScratch w,
                                                                            int limit) {
  constexpr bool DELTA = RULE == kMemoryDelta;
  constexpr int DK = KS * 32, LDK = DK + 8, LDG = DK + 4, LDA = C + 4, VW = 64, LDV = VW + 8;
  constexpr int GB = C * LDG * 4, AB = C * LDA * 4 + C * LDV * 2;
  __shared__ __attribute__((aligned(16))) uint16_t sQ[C * LDK], sK[C * LDK];
  __shared__ __attribute__((aligned(16))) char sX[GB > AB ? GB : AB];
  __shared__ __attribute__((aligned(16))) float tot[4][DK];
  __shared__ float sbeta[C];
  float *sG = reinterpret_cast<float *>(sX), *sA = sG;                       // (one after the other)
  uint16_t *sV = reinterpret_cast<uint16_t *>(sX + C * LDA * 4);
  const PagedSpan *spans = reinterpret_cast<const PagedSpan *>(blob + off_spans);
  const int si = span_of_chunk(spans, num_spans, blockIdx.x);
  if (si < 0) return;
  const PagedSpan sp = spans[si];
  const int t0 = (blockIdx.x - sp.chunk0) * C, h = blockIdx.y, n = min(C, sp.n - t0);
  if (sp.n <= limit) return;
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, l15 = lane & 15;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int hq = h / (a.H / a.G), cols = memory_columns(a);
  const size_t id = (size_t)blockIdx.x * a.H + h, row0 = sp.t0 + t0;
  const size_t slab = (size_t)a.T * a.y.NP, zslab = (size_t)a.T * a.z.NP;

  // queries, keys, log decays: sixteen lanes a row, a wave's sixteen rows; everything is
  // asked for before anything is used
  constexpr int NI = (DK + 127) / 128;
  const f4 nil = {0.f, 0.f, 0.f, 0.f};
  f4 lq[4][NI][2], lk[4][NI][2], lg[4][NI][2];
  uint4 bq[4][NI], bk[4][NI];
  f4 gn[4];  // normed: gates of a row
  float beta = 0.f;
  constexpr int NV = C * VW / 8 / 256;  // 16-byte pieces of a slice of values per thread
  uint4 lv[NV];
  auto fetch_values = [&](int c0) {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int e = tid + i * 256, r = e / (VW / 8), c = c0 + e % (VW / 8) * 8;
      lv[i] = make_uint4(0, 0, 0, 0);
      if (r < n && c < a.vg)
        lv[i] = *reinterpret_cast<const uint4 *>(w.rows + (row0 + r) * cols + 2 * a.G * a.dg + h * a.vg + c);
    }
  };
#pragma unroll
  for (int i4 = 0; i4 < 4; ++i4) {
    const int r = wave * 16 + i4 * 4 + g;
    const size_t t = row0 + min(r, n - 1);
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = min((l15 + 16 * i) * 8, a.dg - 8);
      if constexpr (DELTA) {
        bq[i4][i] = *reinterpret_cast<const uint4 *>(w.rows + t * cols + hq * a.dg + c);
        bk[i4][i] = *reinterpret_cast<const uint4 *>(w.rows + t * cols + (a.G + hq) * a.dg + c);
      } else {
        load8(a.y.p + t * a.y.NP + a.col + hq * a.dg + c, lq[i4][i]);
        load8(a.y.p + t * a.y.NP + a.col + (a.G + hq) * a.dg + c, lk[i4][i]);
      }
      if constexpr (RULE != kMemoryNormed) load8(a.z.p + t * a.z.NP + a.decay.zcol + h * a.dg + c, lg[i4][i]);
    }
    if constexpr (RULE == kMemoryNormed) {
      const float *gt = w.gates + (t * a.H + h) * 3;
      gn[i4] = f4{gt[0], gt[1], 0.f, 0.f};
    }
  }
  if constexpr (DELTA) {
    if (tid < n) beta = a.y.p[(row0 + tid) * a.y.NP + a.col_beta + h];
    fetch_values(0);
  }
  f4 lb[NI][2];
  if constexpr (RULE != kMemoryNormed)
#pragma unroll
    for (int i = 0; i < NI; ++i) load8(a.dbias + (size_t)h * a.dg + min((l15 + 16 * i) * 8, a.dg - 8), lb[i]);
  const float rate = DELTA ? a.rate[h] : 0.f;
  // (products split over K: the other slabs)
  for (int s = 1; s < a.y.S; ++s) {
    if constexpr (DELTA) {
      if (tid < n) beta += a.y.p[s * slab + (row0 + tid) * a.y.NP + a.col_beta + h];
    } else {
#pragma unroll
      for (int i4 = 0; i4 < 4; ++i4)
#pragma unroll
        for (int i = 0; i < NI; ++i) {
          const size_t t = row0 + min(wave * 16 + i4 * 4 + g, n - 1);
          const int c = min((l15 + 16 * i) * 8, a.dg - 8);
          f4 v[2];
          load8(a.y.p + s * slab + t * a.y.NP + a.col + hq * a.dg + c, v);
          lq[i4][i][0] += v[0], lq[i4][i][1] += v[1];
          load8(a.y.p + s * slab + t * a.y.NP + a.col + (a.G + hq) * a.dg + c, v);
          lk[i4][i][0] += v[0], lk[i4][i][1] += v[1];
        }
    }
  }
  if constexpr (RULE != kMemoryNormed)
    for (int s = 1; s < a.z.S; ++s)
#pragma unroll
      for (int i4 = 0; i4 < 4; ++i4)
#pragma unroll
        for (int i = 0; i < NI; ++i) {
          f4 v[2];
          load8(a.z.p + s * zslab + (row0 + min(wave * 16 + i4 * 4 + g, n - 1)) * a.z.NP + a.decay.zcol + h * a.dg +
                    min((l15 + 16 * i) * 8, a.dg - 8), v);
          lg[i4][i][0] += v[0], lg[i4][i][1] += v[1];
        }
  if constexpr (DELTA)
    if (tid < C) sbeta[tid] = tid < n ? sigmoid_f(beta) : 0.f;
#pragma unroll
  for (int i4 = 0; i4 < 4; ++i4) {
    const int r = wave * 16 + i4 * 4 + g;
    const bool real = r < n;
    f4 q[NI][2], k[NI][2];
    float qq = 0.f, kk = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      if constexpr (DELTA) {
        unpack8_bf16(bq[i4][i], q[i][0], q[i][1]);
        unpack8_bf16(bk[i4][i], k[i][0], k[i][1]);
      } else {
#pragma unroll
        for (int j = 0; j < 2; ++j) q[i][j] = lq[i4][i][j], k[i][j] = lk[i4][i][j];
      }
      if (!real || (l15 + 16 * i) * 8 >= a.dg) q[i][0] = q[i][1] = k[i][0] = k[i][1] = nil;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        qq = fmaf(q[i][e >> 2][e & 3], q[i][e >> 2][e & 3], qq);
        kk = fmaf(k[i][e >> 2][e & 3], k[i][e >> 2][e & 3], kk);
      }
    }
    float fq = a.q_scale, fk = 1.f;
    if (a.unit) {
#pragma unroll
      for (int o = 1; o < 16; o <<= 1) qq += __shfl_xor(qq, o), kk += __shfl_xor(kk, o);
      fq *= __fdiv_rn(1.0f, sqrtf(qq + 1e-6f)), fk = __fdiv_rn(1.0f, sqrtf(kk + 1e-6f));
    }
    if constexpr (RULE == kMemoryNormed) fk = ex2(gn[i4][1]);
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (l15 + 16 * i) * 8;
      if (c >= DK) continue;
      *reinterpret_cast<uint4 *>(&sQ[r * LDK + c]) = pack8_bf16(q[i][0] * fq, q[i][1] * fq);
      *reinterpret_cast<uint4 *>(&sK[r * LDK + c]) = pack8_bf16(k[i][0] * fk, k[i][1] * fk);
      f4 d[2];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        float v = 0.f;
        if constexpr (RULE == kMemoryNormed) v = gn[i4][0];
        else v = c + e < a.dim ? log2_decay<RULE>(a, rate, lg[i4][i][e >> 2][e & 3] + lb[i][e >> 2][e & 3]) : 0.f;
        d[e >> 2][e & 3] = real ? v : 0.f;
      }
      *reinterpret_cast<f4 *>(&sG[r * LDG + c]) = d[0], *reinterpret_cast<f4 *>(&sG[r * LDG + c + 4]) = d[1];
    }
  }
  __syncthreads();
  // sums of the log decays within the wave's block
#pragma unroll
  for (int i = 0; i < (DK + 63) / 64; ++i) {
    const int c = lane + 64 * i;
    if (c >= DK) continue;
    float s = 0.f;
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      float *p = &sG[(wave * 16 + r) * LDG + c];
      s += *p;
      *p = s;
    }
    tot[wave][c] = s;
  }
  __syncthreads();

  // scores: lane = (token i of the wave's block, 4 tokens j of a block)
  bool narrow = true;
  for (int c = lane; c < DK; c += 64) narrow = narrow && tot[wave][c] > -kSpread;
  narrow = __all(narrow);
  const int ri = wave * 16 + l15;
  f4 sq[4], sk[4];
#pragma unroll
  for (int b = 0; b < 4; ++b) sq[b] = sk[b] = f4{0.f, 0.f, 0.f, 0.f};
  uint4 kd[KS];  // k_j exp(G_last - G_j)
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) {
    const int c = ks * 32 + 8 * g;
    f4 q[2], k[2], gi[2], fi[2];
    unpack8_bf16(*reinterpret_cast<const uint4 *>(&sQ[ri * LDK + c]), q[0], q[1]);
    unpack8_bf16(*reinterpret_cast<const uint4 *>(&sK[ri * LDK + c]), k[0], k[1]);
    gi[0] = *reinterpret_cast<const f4 *>(&sG[ri * LDG + c]), gi[1] = *reinterpret_cast<const f4 *>(&sG[ri * LDG + c + 4]);
#pragma unroll
    for (int e = 0; e < 8; ++e) fi[e >> 2][e & 3] = ex2(gi[e >> 2][e & 3]);
    const auto times = [](const f4 (&x)[2], const f4 (&y)[2]) {
      return __builtin_bit_cast(bf8, pack8_bf16(x[0] * y[0], x[1] * y[1]));
    };
    if (narrow) {
      f4 inv[2];
#pragma unroll
      for (int e = 0; e < 8; ++e) inv[e >> 2][e & 3] = ex2(-gi[e >> 2][e & 3]);
      const bf8 kj = times(k, inv);
#pragma unroll
      for (int b = 0; b < 4; ++b)
        if (b == wave) {
          sq[b] = mma(kj, times(q, fi), sq[b]);
          if constexpr (DELTA) sk[b] = mma(kj, times(k, fi), sk[b]);
        }
    }
#pragma unroll
    for (int b = 2; b >= 0; --b) {
      if (b >= wave) continue;
      f4 x[2], gj[2], tb[2];
      const int rj = b * 16 + l15;
      tb[0] = *reinterpret_cast<const f4 *>(&tot[b][c]), tb[1] = *reinterpret_cast<const f4 *>(&tot[b][c + 4]);
      gj[0] = *reinterpret_cast<const f4 *>(&sG[rj * LDG + c]), gj[1] = *reinterpret_cast<const f4 *>(&sG[rj * LDG + c + 4]);
      unpack8_bf16(*reinterpret_cast<const uint4 *>(&sK[rj * LDK + c]), x[0], x[1]);
#pragma unroll
      for (int e = 0; e < 8; ++e) gj[e >> 2][e & 3] = ex2(tb[e >> 2][e & 3] - gj[e >> 2][e & 3]);
      const bf8 kj = times(x, gj);
      sq[b] = mma(kj, times(q, fi), sq[b]);
      if constexpr (DELTA) sk[b] = mma(kj, times(k, fi), sk[b]);
#pragma unroll
      for (int e = 0; e < 8; ++e) fi[e >> 2][e & 3] *= ex2(tb[e >> 2][e & 3]);
    }
    // fi: exp(G_i) from the chunk's start
    *reinterpret_cast<uint4 *>(w.qg + (id * C + ri) * DK + c) = pack8_bf16(q[0] * fi[0], q[1] * fi[1]);
    f4 rest[2];
    rest[0] = *reinterpret_cast<const f4 *>(&tot[wave][c]) - gi[0], rest[1] = *reinterpret_cast<const f4 *>(&tot[wave][c + 4]) - gi[1];
#pragma unroll
    for (int b = 1; b < 4; ++b)
      if (b > wave) rest[0] += *reinterpret_cast<const f4 *>(&tot[b][c]), rest[1] += *reinterpret_cast<const f4 *>(&tot[b][c + 4]);
#pragma unroll
    for (int e = 0; e < 8; ++e) rest[e >> 2][e & 3] = ex2(rest[e >> 2][e & 3]);
    kd[ks] = pack8_bf16(k[0] * rest[0], k[1] * rest[1]);
    if constexpr (DELTA)  // (this row of sQ is the wave's own)
      if (narrow) *reinterpret_cast<uint4 *>(&sQ[ri * LDK + c]) = pack8_bf16(k[0] * fi[0], k[1] * fi[1]);
  }
  if (!narrow) {  // pair by pair
    f4 dq = f4{0.f, 0.f, 0.f, 0.f}, dk = dq;
    for (int c = 0; c < DK; ++c) {
      const float q = bf2f(sQ[ri * LDK + c]), k = bf2f(sK[ri * LDK + c]), gi = sG[ri * LDG + c];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int j = wave * 16 + 4 * g + e;
        const float f = bf2f(sK[j * LDK + c]) * ex2(fminf(gi - sG[j * LDG + c], 0.f));
        dq[e] = fmaf(q, f, dq[e]), dk[e] = fmaf(k, f, dk[e]);
      }
    }
#pragma unroll
    for (int b = 0; b < 4; ++b)
      if (b == wave) sq[b] = dq, sk[b] = dk;
    if constexpr (DELTA) {
      for (int ks = 0; ks < KS; ++ks) {
        const int c = ks * 32 + 8 * g;
        f4 k[2], gi[2];
        unpack8_bf16(*reinterpret_cast<const uint4 *>(&sK[ri * LDK + c]), k[0], k[1]);
        gi[0] = *reinterpret_cast<const f4 *>(&sG[ri * LDG + c]), gi[1] = *reinterpret_cast<const f4 *>(&sG[ri * LDG + c + 4]);
#pragma unroll
        for (int b = 0; b < 3; ++b)
          if (b < wave) gi[0] += *reinterpret_cast<const f4 *>(&tot[b][c]), gi[1] += *reinterpret_cast<const f4 *>(&tot[b][c + 4]);
#pragma unroll
        for (int e = 0; e < 8; ++e) gi[e >> 2][e & 3] = ex2(gi[e >> 2][e & 3]);
        *reinterpret_cast<uint4 *>(&sQ[ri * LDK + c]) = pack8_bf16(k[0] * gi[0], k[1] * gi[1]);
      }
    }
  }
#pragma unroll
  for (int b = 0; b < 4; ++b) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int j = b * 16 + 4 * g + e;
      if (j > ri) sq[b][e] = 0.f;
      if (j >= ri) sk[b][e] = 0.f;
    }
    *reinterpret_cast<uint2 *>(w.p + (id * C + ri) * C + b * 16 + 4 * g) = pack4(sq[b]);
  }
  for (int c = tid; c < DK; c += 256) w.last[id * DK + c] = ex2(tot[0][c] + tot[1][c] + tot[2][c] + tot[3][c]);
  __syncthreads();  // (keys and sums of decays are read)
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) *reinterpret_cast<uint4 *>(&sK[ri * LDK + ks * 32 + 8 * g]) = kd[ks];
  if constexpr (DELTA) {
    const float beta = sbeta[ri];
#pragma unroll
    for (int b = 0; b < 4; ++b)
      if (b <= wave) *reinterpret_cast<f4 *>(&sA[ri * LDA + b * 16 + 4 * g]) = sk[b] * beta;
  }
  __syncthreads();
  for (int ct = wave; ct < 2 * KS; ct += 4)
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
      *reinterpret_cast<bf8 *>(w.kd + (id * DK + ct * 16 + l15) * C + kb * 32 + 8 * g) = read_columns<LDK>(sK, kb, ct * 16);

  if constexpr (DELTA) {
    // T in A's place.  Its blocks on the diagonal: a lane has a column, rows in turn
    {
      float x[16];
      const float *A = &sA[wave * 16 * LDA + wave * 16];
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        float v = i == l15 ? 1.f : 0.f;
#pragma unroll
        for (int j = 0; j < 16; ++j)
          if (j < i) v = fmaf(-A[i * LDA + j], x[j], v);
        x[i] = v;
      }
      __syncthreads();
      if (g == 0)
#pragma unroll
        for (int i = 0; i < 16; ++i) sA[(wave * 16 + i) * LDA + wave * 16 + l15] = x[i];
      __syncthreads();
    }
    // the rows of blocks below, from the top: T_ij = -T_ii sum over k of A_ik T_kj
#pragma unroll
    for (int i = 1; i < 4; ++i) {
      f4 x = f4{0.f, 0.f, 0.f, 0.f}, y = x;
      if (wave < i) {
        for (int k = wave; k < i; ++k)
#pragma unroll
          for (int s = 0; s < 4; ++s)
            x = __builtin_amdgcn_mfma_f32_16x16x4f32(sA[(i * 16 + l15) * LDA + k * 16 + s * 4 + g],
                                                     sA[(k * 16 + s * 4 + g) * LDA + wave * 16 + l15], x, 0, 0, 0);
#pragma unroll
        for (int s = 0; s < 4; ++s)  // (x: rows 4g + s of column l15, as it stands)
          y = __builtin_amdgcn_mfma_f32_16x16x4f32(sA[(i * 16 + l15) * LDA + i * 16 + 4 * g + s], x[s], y, 0, 0, 0);
      }
      __syncthreads();
      if (wave < i)
#pragma unroll
        for (int e = 0; e < 4; ++e) sA[(i * 16 + 4 * g + e) * LDA + wave * 16 + l15] = -y[e];
      __syncthreads();
    }
    // this wave's rows of T, times beta: value and remainder
    bf8 th[2], tl[2];
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int j = kb * 32 + 8 * g + e;
        __bf16 hi, lo;
        split2((j >> 4) <= wave ? sA[ri * LDA + j] * sbeta[j] : 0.f, hi, lo);
        th[kb][e] = hi, tl[kb][e] = lo;
      }
#pragma unroll
    for (int ct = 0; ct < 2 * KS; ++ct) {
      f4 x = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
        if (kb * 2 > wave) continue;
        const bf8 kg = read_columns<LDK>(sQ, kb, ct * 16);
        x = mma(kg, th[kb], x);
        x = mma(kg, tl[kb], x);
      }
      *reinterpret_cast<uint2 *>(w.w + (id * C + ri) * DK + ct * 16 + 4 * g) = pack4(x);
    }
    for (int c0 = 0; c0 < a.vs; c0 += VW) {
      __syncthreads();
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int e = tid + i * 256;
        *reinterpret_cast<uint4 *>(&sV[e / (VW / 8) * LDV + e % (VW / 8) * 8]) = lv[i];
      }
      if (c0 + VW < a.vs) fetch_values(c0 + VW);
      __syncthreads();
#pragma unroll
      for (int ct = 0; ct < VW / 16; ++ct) {
        if (c0 + ct * 16 >= a.vs) continue;
        f4 x = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) {
          if (kb * 2 > wave) continue;
          const bf8 v = read_columns<LDV>(sV, kb, ct * 16);
          x = mma(v, th[kb], x);
          x = mma(v, tl[kb], x);
        }
        *reinterpret_cast<f4 *>(w.u + (id * C + ri) * a.vs + c0 + ct * 16 + 4 * g) = x;
      }
    }
  }
}

// The pass over the chunks: a workgroup per (head, VS state columns, span); a head's are
// mostly on one XCD, which then reads the chunk's operands once.  Wave w: rows
// 16 w .. of u and o, and of the state 16 columns and an even share of the rows, in
// registers (lane: 4 rows of one column); the state goes to LDS once a chunk as the
// operand [column][row], u as rows.  What the next chunk needs is fetched a chunk ahead.
template <MemoryRule RULE, int KS, int VS>
__global__ __launch_bounds__(256, KS * VS <= (RULE == kMemoryDelta ? 64 : 128) ? 2 : 1) void memory_scan_kernel(const char *__restrict__ blob, int off_spans,
                                                                           Memory a, MemoryScratch w, int limit) {
  constexpr bool DELTA = RULE == kMemoryDelta;
  constexpr int DK = KS * 32, LDK = DK + 8, LDU = VS + 8;
  constexpr int VT = VS / 16, WD = 4 / VT, ND = (2 * KS + WD - 1) / WD;
  __shared__ __attribute__((aligned(16))) uint16_t sHi[VS * LDK], sLo[VS * LDK], sU[C * LDU], sUl[DELTA ? C * LDU : 8];
  const PagedSpan sp = reinterpret_cast<const PagedSpan *>(blob + off_spans)[blockIdx.z];
  if (sp.n <= limit) return;
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, l15 = lane & 15;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x, c0 = blockIdx.y * VS, vw = min(VS, a.vs - c0);
  const int ri = wave * 16 + l15, vcol = wave % VT * 16 + l15, d0 = wave / VT * ND;
  const size_t id0 = (size_t)sp.chunk0 * a.H + h;

  bf8 fq[KS], fw[DELTA ? KS : 1], fp[2], fk[ND][2];
  f4 fu[VT], fl[ND];
  auto fetch = [&](int chunk) {
    const size_t id = id0 + (size_t)chunk * a.H;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const size_t at = (id * C + ri) * DK + ks * 32 + 8 * g;
      if constexpr (DELTA) fw[ks] = *reinterpret_cast<const bf8 *>(w.w + at);
      fq[ks] = *reinterpret_cast<const bf8 *>(w.qg + at);
    }
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) {
      const int c = c0 + min(vt * 16, vw - 16) + 4 * g;
      if constexpr (DELTA) {
        fu[vt] = *reinterpret_cast<const f4 *>(w.u + (id * C + ri) * a.vs + c);
      } else {  // the values as the product left them
        fu[vt] = f4{0.f, 0.f, 0.f, 0.f};
        const int t = chunk * C + ri;
        if (t < sp.n && c < a.vg) {
          const float *p = a.y.p + (size_t)(sp.t0 + t) * a.y.NP + a.col + 2 * a.G * a.dg + h * a.vg + c;
          fu[vt] = *reinterpret_cast<const f4 *>(p);
          for (int s = 1; s < a.y.S; ++s) fu[vt] += *reinterpret_cast<const f4 *>(p + (size_t)s * a.T * a.y.NP);
        }
        if constexpr (RULE == kMemoryNormed)
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (c + e == a.vdim && t < sp.n) fu[vt][e] = 1.f;
      }
    }
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) fp[kb] = *reinterpret_cast<const bf8 *>(w.p + (id * C + ri) * C + kb * 32 + 8 * g);
#pragma unroll
    for (int dt = 0; dt < ND; ++dt) {
      const int tile = min(d0 + dt, 2 * KS - 1);
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
        fk[dt][kb] = *reinterpret_cast<const bf8 *>(w.kd + (id * DK + tile * 16 + l15) * C + kb * 32 + 8 * g);
      fl[dt] = *reinterpret_cast<const f4 *>(w.last + id * DK + tile * 16 + 4 * g);
    }
  };
  fetch(0);
  f4 st[ND];
  float *S = a.state + (((size_t)sp.slot * a.H + h) * a.dg) * a.vs + c0 + vcol;
#pragma unroll
  for (int dt = 0; dt < ND; ++dt) {
    st[dt] = f4{0.f, 0.f, 0.f, 0.f};
    if (sp.pos0 > 0 && (d0 + dt) * 16 < a.dg && vcol < vw)
#pragma unroll
      for (int e = 0; e < 4; ++e) st[dt][e] = S[(size_t)((d0 + dt) * 16 + 4 * g + e) * a.vs];
  }
  auto publish = [&]() {
#pragma unroll
    for (int dt = 0; dt < ND; ++dt) {
      if (2 * KS % WD && d0 + dt >= 2 * KS) continue;
      f4 lo;
#pragma unroll
      for (int e = 0; e < 4; ++e) lo[e] = st[dt][e] - (float)(__bf16)st[dt][e];
      const int at = vcol * LDK + (d0 + dt) * 16 + 4 * g;
      *reinterpret_cast<uint2 *>(&sHi[at]) = pack4(st[dt]);
      *reinterpret_cast<uint2 *>(&sLo[at]) = pack4(lo);
    }
  };
  publish();
  for (int chunk = 0; chunk * C < sp.n; ++chunk) {
    __syncthreads();
    f4 o[VT], olo[VT], u[VT], ulo[VT];
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) o[vt] = olo[vt] = u[vt] = ulo[vt] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) {
        const int at = (vt * 16 + l15) * LDK + ks * 32 + 8 * g;
        const bf8 hi = *reinterpret_cast<const bf8 *>(&sHi[at]), lo = *reinterpret_cast<const bf8 *>(&sLo[at]);
        if constexpr (DELTA) {
          u[vt] = mma(hi, fw[ks], u[vt]);
          ulo[vt] = mma(lo, fw[ks], ulo[vt]);
        }
        o[vt] = mma(hi, fq[ks], o[vt]);
        olo[vt] = mma(lo, fq[ks], olo[vt]);
      }
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) {
      const int at = ri * LDU + vt * 16 + 4 * g;
      if constexpr (DELTA) {
        u[vt] = fu[vt] - u[vt] - ulo[vt];
        f4 lo;
#pragma unroll
        for (int e = 0; e < 4; ++e) lo[e] = u[vt][e] - (float)(__bf16)u[vt][e];
        *reinterpret_cast<uint2 *>(&sU[at]) = pack4(u[vt]);
        *reinterpret_cast<uint2 *>(&sUl[at]) = pack4(lo);
      } else {
        *reinterpret_cast<uint2 *>(&sU[at]) = pack4(fu[vt]);
      }
      o[vt] += olo[vt];
    }
    bf8 p[2], k[ND][2];
    f4 last[ND];
    p[0] = fp[0], p[1] = fp[1];
#pragma unroll
    for (int dt = 0; dt < ND; ++dt) k[dt][0] = fk[dt][0], k[dt][1] = fk[dt][1], last[dt] = fl[dt];
    if ((chunk + 1) * C < sp.n) fetch(chunk + 1);
    __syncthreads();
#pragma unroll
    for (int dt = 0; dt < ND; ++dt) st[dt] *= last[dt];
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      if (kb * 2 <= wave)
#pragma unroll
        for (int vt = 0; vt < VT; ++vt) {
          o[vt] = mma(read_columns<LDU>(sU, kb, vt * 16), p[kb], o[vt]);
          if constexpr (DELTA) o[vt] = mma(read_columns<LDU>(sUl, kb, vt * 16), p[kb], o[vt]);
        }
      const bf8 uh = read_columns<LDU>(sU, kb, wave % VT * 16);
#pragma unroll
      for (int dt = 0; dt < ND; ++dt) st[dt] = mma(k[dt][kb], uh, st[dt]);
      if constexpr (DELTA) {
        const bf8 ul = read_columns<LDU>(sUl, kb, wave % VT * 16);
#pragma unroll
        for (int dt = 0; dt < ND; ++dt) st[dt] = mma(k[dt][kb], ul, st[dt]);
      }
    }
    if (chunk * C + ri < sp.n) {
      float *dst = w.o + ((size_t)(sp.t0 + chunk * C + ri) * a.H + h) * a.vs + c0 + 4 * g;
#pragma unroll
      for (int vt = 0; vt < VT; ++vt)
        if (vt * 16 < vw) *reinterpret_cast<f4 *>(dst + vt * 16) = o[vt];
    }
    if ((chunk + 1) * C < sp.n) publish();
  }
#pragma unroll
  for (int dt = 0; dt < ND; ++dt)
    if ((d0 + dt) * 16 < a.dg && vcol < vw)
#pragma unroll
      for (int e = 0; e < 4; ++e) S[(size_t)((d0 + dt) * 16 + 4 * g + e) * a.vs] = st[dt][e];
}

// norm and gate: sixteen lanes a (token, head), their columns 64 apart
template <MemoryRule RULE>
__global__ __launch_bounds__(256) void memory_out_kernel(const char *__restrict__ blob, Memory a, MemoryScratch w,
                                                         int above) {
  const int l15 = threadIdx.x & 15;
  const long id = blockIdx.x * 16L + (threadIdx.x >> 4);
  const int t = (int)min(id / a.H, (long)a.T - 1), h = (int)(id % a.H);
  const PagedToken tk = reinterpret_cast<const PagedToken *>(blob + a.off_tokens)[t];
  const bool mine = id < (long)a.T * a.H && tk.back + tk.ahead + 1 > above;
  const float *o = w.o + ((size_t)t * a.H + h) * a.vs;
  const bool second = a.gate.r > 0;
  const Partials &gp = second ? a.z : a.y;
  const size_t gat = (size_t)t * gp.NP + (second ? a.gate.zcol : a.col_gate) + h * a.vg;
  constexpr int NK = 2;  // pieces of 8 columns kept in registers
  f4 v[NK][2], gt[NK][2];
  float f = 1.f, ss = 0.f;
  if (mine) {
#pragma unroll
    for (int k = 0; k < NK; ++k) {
      const int c = min(l15 * 8 + k * 128, a.vg - 8);
      load8(o + c, v[k]);
      sum8(gp, (size_t)a.T * gp.NP, gat + c, gt[k]);
    }
    if constexpr (RULE == kMemoryNormed)
      f = __fdiv_rn(1.0f, fmaxf(fabsf(o[a.vdim]), expf(-w.gates[((size_t)t * a.H + h) * 3 + 2])) + 1e-6f);
    auto add = [&](const f4 (&x)[2], int c) {
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float y = x[e >> 2][e & 3] * f;
        if (c + e < a.vdim) ss = fmaf(y, y, ss);
      }
    };
#pragma unroll
    for (int k = 0; k < NK; ++k) add(v[k], l15 * 8 + k * 128);
    for (int c = l15 * 8 + NK * 128; c < a.vg; c += 128) {
      f4 x[2];
      load8(o + c, x);
      add(x, c);
    }
  }
#pragma unroll
  for (int k = 1; k < 16; k <<= 1) ss += __shfl_xor(ss, k);
  if (!mine) return;
  const float r = f * inv_rms(ss, a.vdim, a.eps);
  auto put = [&](f4 (&x)[2], const f4 (&y)[2], int c) {
    f4 wv[2];
    load8(a.norm + (a.norm_heads ? h * a.vg : 0) + c, wv);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float gv = y[e >> 2][e & 3], sg = __builtin_amdgcn_rcpf(1.f + ex2(-kLog2e * gv));
      const float z = x[e >> 2][e & 3] * r * wv[e >> 2][e & 3] * (a.gate_silu ? gv * sg : sg);
      x[e >> 2][e & 3] = c + e < a.vdim ? z : 0.f;
    }
    *reinterpret_cast<uint4 *>((uint16_t *)a.out + act_packed_off(t, a.out_col + h * a.vg + c, a.ldo)) = pack8_bf16(x[0], x[1]);
  };
#pragma unroll
  for (int k = 0; k < NK; ++k)
    if (l15 * 8 + k * 128 < a.vg) put(v[k], gt[k], l15 * 8 + k * 128);
  for (int c = l15 * 8 + NK * 128; c < a.vg; c += 128) {
    f4 x[2], y[2];
    load8(o + c, x);
    sum8(gp, (size_t)a.T * gp.NP, gat + c, y);
    put(x, y, c);
  }
}

template <MemoryRule RULE>
hipError_t run_chunks(const char *blob, int off_spans, int num_spans, int num_chunks, const Memory &a,
                      const MemoryScratch &w, int limit, hipStream_t s) {
  if (RULE == kMemoryNormed)
    hipLaunchKernelGGL(memory_gates_kernel, dim3(a.H, num_spans), dim3(256), 0, s, blob, off_spans, a, w, limit);
  if (RULE == kMemoryDelta) {
    ConvRows c;
    c.u = a.y, c.T = a.T, c.col = a.col, c.cols = 2 * a.G * a.dg + a.H * a.vg, c.taps = a.taps, c.conv = a.conv;
    c.carry = a.carry, c.silu = a.silu, c.hb = w.rows, c.off_tokens = a.off_tokens, c.above = limit;
    if (const hipError_t e = launch_conv_rows(blob, c, s)) return e;
  }
  // narrow workgroups where the spans and heads alone do not fill the chip
  const bool wide = (long)a.H * num_spans * (a.vs / 16) > 512;
#define FFMI_MS(KS, VS)                                                                                             \
  hipLaunchKernelGGL((memory_scan_kernel<RULE, KS, VS>), dim3(a.H, (a.vs + VS - 1) / VS, num_spans), dim3(256), 0, s, \
                     blob, off_spans, a, w, limit)
#define FFMI_MC(KS)                                                                                              \
  do {                                                                                                           \
    hipLaunchKernelGGL((memory_chunk_kernel<RULE, KS>), dim3(num_chunks, a.H), dim3(256), 0, s, blob, off_spans, \
                       num_spans, a, w, limit);                                                                  \
    if (wide) FFMI_MS(KS, 32);                                                                                   \
    else FFMI_MS(KS, 16);                                                                                        \
  } while (0)
  switch (memory_chunk_width(a.dg)) {
    case 32: FFMI_MC(1); break;
    case 64: FFMI_MC(2); break;
    case 128: FFMI_MC(4); break;
    default: FFMI_MC(8); break;
  }
#undef FFMI_MC
#undef FFMI_MS
  return hipGetLastError();
}

}  // namespace

hipError_t launch_memory_chunks(const char *blob, int off_spans, int num_spans, int num_chunks, const Memory &a,
                                const MemoryScratch &w, int limit, hipStream_t s) {
  if (num_spans <= 0 || num_chunks <= 0) return hipSuccess;
  if (a.H < 1 || a.G < 1 || a.H % a.G || a.dg % 32 || a.vg % 32 || a.dg > kMemoryMaxChunkDim || a.dim > a.dg ||
      a.vdim > a.vg || a.vs != memory_state_columns(a.rule, a.vdim) || a.y.S < 1 || a.y.NP % 4 || a.col % 4 ||
      a.decay.zcol % 4 || limit < a.taps || limit < kShortSpan || (a.rule == kMemoryDelta) != (a.taps > 0) ||
      (a.taps > 0 && !a.conv) || (a.taps > 1 && !a.carry) ||
      (a.rule != kMemoryNormed && (a.z.S < 1 || a.z.NP % 4 || !a.dbias)) || !w.qg || !w.kd || !w.p || !w.last ||
      !w.o || (a.rule == kMemoryDelta && (!w.w || !w.u || !w.rows || !a.rate)) ||
      (a.rule == kMemoryNormed && !w.gates) || num_chunks > 65535)
    return hipErrorInvalidValue;
  if (a.rule == kMemoryGated) return run_chunks<kMemoryGated>(blob, off_spans, num_spans, num_chunks, a, w, limit, s);
  if (a.rule == kMemoryDelta) return run_chunks<kMemoryDelta>(blob, off_spans, num_spans, num_chunks, a, w, limit, s);
  return run_chunks<kMemoryNormed>(blob, off_spans, num_spans, num_chunks, a, w, limit, s);
}

hipError_t launch_memory_out(const char *blob, const Memory &a, const MemoryScratch &w, int above, hipStream_t s) {
  if (a.T <= 0) return hipSuccess;
  if (!w.o || (a.rule == kMemoryNormed && !w.gates) || a.vg % 32 || a.ldo % 32 || a.out_col % 32 || a.col_gate % 4 ||
      a.gate.zcol % 4 || (a.gate.r > 0 && a.z.S < 1) || a.out_col + a.H * a.vg > a.ldo)
    return hipErrorInvalidValue;
  const dim3 grid((unsigned)(((long)a.T * a.H + 15) / 16));
#define FFMI_MO(RULE) hipLaunchKernelGGL(memory_out_kernel<RULE>, grid, dim3(256), 0, s, blob, a, w, above)
  if (a.rule == kMemoryGated) FFMI_MO(kMemoryGated);
  else if (a.rule == kMemoryDelta) FFMI_MO(kMemoryDelta);
  else FFMI_MO(kMemoryNormed);
#undef FFMI_MO
  return hipGetLastError();
}

}  // namespace ffmi
