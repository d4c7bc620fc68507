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
// The first launch makes what does not need S, all chunks side by side; the second passes
// over a span's chunks with the state in registers; the third has the outputs' norm and gate.
//
// No exponent is ever positive beyond kSpread: a chunk's four blocks of 16 tokens take their
// decays from the blocks' borders, and a block's own 16 x 16 products from its start while
// its decays add up to less than that, else one exponential per pair and channel.
// Logs of decays have base 2.
#include <algorithm>

#include "memory_util.h"

namespace ffmi {

namespace {

typedef short s4 __attribute__((ext_vector_type(4)));
constexpr int C = kMemoryChunk;
constexpr float kLog2e = 1.4426950408889634f;
constexpr float kSpread = 80.f;  // base 2: far from fp32's and bf16's range on either side

__device__ __forceinline__ float ex2(float v) { return __builtin_amdgcn_exp2f(v); }
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

// columns c .. c + 7 of q | k | v for token t of the span, convolved
__device__ __forceinline__ void project8(const Memory &a, const PagedSpan &sp, int bank, int t, int c, bool keep,
                                         f4 (&v)[2]) {
  const size_t slab = (size_t)a.T * a.y.NP, at = (size_t)(sp.t0 + t) * a.y.NP + a.col + c;
  sum8(a.y, slab, at, v);
  if (a.taps > 0) {
    const size_t cols = memory_columns(a);
    const int past = a.taps - 1;
    const float *old = a.carry + ((size_t)sp.slot * 2 + bank) * past * cols + c;
    if (keep && sp.n - 1 - t < past) {  // (spans of this form are longer than that)
      float *now = a.carry + ((size_t)sp.slot * 2 + (bank ^ 1)) * past * cols + (sp.n - 1 - t) * cols + c;
      *reinterpret_cast<f4 *>(now) = v[0], *reinterpret_cast<f4 *>(now + 4) = v[1];
    }
    const float *w = a.conv + c;
    v[0] *= *reinterpret_cast<const f4 *>(w + past * cols), v[1] *= *reinterpret_cast<const f4 *>(w + past * cols + 4);
    for (int d = 1; d <= past && d <= sp.pos0 + t; ++d) {
      f4 u[2];
      if (t >= d) {
        sum8(a.y, slab, at - (size_t)d * a.y.NP, u);
      } else {
        const float *o = old + (d - t - 1) * cols;
        u[0] = *reinterpret_cast<const f4 *>(o), u[1] = *reinterpret_cast<const f4 *>(o + 4);
      }
      const float *wd = w + (past - d) * cols;
      v[0] += u[0] * *reinterpret_cast<const f4 *>(wd), v[1] += u[1] * *reinterpret_cast<const f4 *>(wd + 4);
    }
  }
  if (a.silu)
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e >> 2][e & 3] = silu_f(v[e >> 2][e & 3]);
}

// normed: decay, key factor (logs, base 2) and m of every token of a long span; a workgroup
// per (head, span), m by a scan of the maps m -> max(m + f, i)
__global__ __launch_bounds__(256) void memory_gates_kernel(const char *__restrict__ blob, int off_spans, Memory a,
                                                           MemoryScratch w, int limit) {
  __shared__ float sa[2][256], sb[2][256];
  const PagedSpan sp = reinterpret_cast<const PagedSpan *>(blob + off_spans)[blockIdx.y];
  if (sp.n <= limit) return;
  const int tid = threadIdx.x, h = blockIdx.x, per = (sp.n + 255) / 256;
  const int b = min(tid * per, sp.n), e = min(b + per, sp.n);
  const int bank = reinterpret_cast<const PagedToken *>(blob + a.off_tokens)[sp.t0].bank;
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

// A workgroup per (chunk, head, span); wave b has the chunk's block of 16 tokens b.
template <MemoryRule RULE, int KS>
__global__ __launch_bounds__(256) void memory_chunk_kernel(const char *__restrict__ blob, int off_spans, Memory a,
                                                           MemoryScratch w, int limit) {
  constexpr bool DELTA = RULE == kMemoryDelta;
  constexpr int DK = KS * 32, LDK = DK + 8, LDG = DK + 4, LDA = C + 4, VW = 64, LDV = VW + 8;
  constexpr int GB = C * LDG * 4, AB = C * LDA * 4 + C * LDV * 2;
  __shared__ __attribute__((aligned(16))) uint16_t sQ[C * LDK], sK[C * LDK];
  __shared__ __attribute__((aligned(16))) char sX[GB > AB ? GB : AB];
  __shared__ __attribute__((aligned(16))) float tot[4][DK];
  __shared__ float sbeta[C];
  float *sG = reinterpret_cast<float *>(sX), *sA = sG;                       // (one after the other)
  uint16_t *sV = reinterpret_cast<uint16_t *>(sX + C * LDA * 4);
  const PagedSpan sp = reinterpret_cast<const PagedSpan *>(blob + off_spans)[blockIdx.z];
  const int t0 = blockIdx.x * C, h = blockIdx.y, n = min(C, sp.n - t0);
  if (sp.n <= limit || n <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, l15 = lane & 15;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int bank = reinterpret_cast<const PagedToken *>(blob + a.off_tokens)[sp.t0].bank;
  const int hq = h / (a.H / a.G);
  const bool first = h % (a.H / a.G) == 0;  // (query and key heads are shared)
  const size_t id = ((size_t)(sp.t0 / C) + blockIdx.z + blockIdx.x) * a.H + h;

  // queries, keys, log decays: sixteen lanes a row
  constexpr int NI = (DK + 127) / 128;
  for (int r4 = 0; r4 < 16; r4 += 4) {
    const int r = wave * 16 + r4 + g, t = t0 + r;
    const bool real = r < n;
    f4 q[NI][2], k[NI][2];
    float qq = 0.f, kk = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (l15 + 16 * i) * 8;
#pragma unroll
      for (int j = 0; j < 2; ++j) q[i][j] = k[i][j] = f4{0.f, 0.f, 0.f, 0.f};
      if (real && c < a.dg) {
        project8(a, sp, bank, t, hq * a.dg + c, first, q[i]);
        project8(a, sp, bank, t, (a.G + hq) * a.dg + c, first, k[i]);
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        qq = fmaf(q[i][e >> 2][e & 3], q[i][e >> 2][e & 3], qq);
        kk = fmaf(k[i][e >> 2][e & 3], k[i][e >> 2][e & 3], kk);
      }
    }
    float fq = a.q_scale, fk = 1.f, gs = 0.f;
    if (a.unit) {
#pragma unroll
      for (int o = 1; o < 16; o <<= 1) qq += __shfl_xor(qq, o), kk += __shfl_xor(kk, o);
      fq *= __fdiv_rn(1.0f, sqrtf(qq + 1e-6f)), fk = __fdiv_rn(1.0f, sqrtf(kk + 1e-6f));
    }
    if constexpr (RULE == kMemoryNormed)
      if (real) {
        const float *gt = w.gates + ((size_t)(sp.t0 + t) * a.H + h) * 3;
        gs = gt[0], fk = ex2(gt[1]);
      }
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = (l15 + 16 * i) * 8;
      if (c >= DK) continue;
      *reinterpret_cast<uint4 *>(&sQ[r * LDK + c]) = pack8_bf16(q[i][0] * fq, q[i][1] * fq);
      *reinterpret_cast<uint4 *>(&sK[r * LDK + c]) = pack8_bf16(k[i][0] * fk, k[i][1] * fk);
      f4 d[2];
      d[0] = d[1] = f4{gs, gs, gs, gs};
      if constexpr (RULE != kMemoryNormed)
        if (real && c < a.dg) {
          sum8(a.z, (size_t)a.T * a.z.NP, (size_t)(sp.t0 + t) * a.z.NP + a.decay.zcol + h * a.dg + c, d);
#pragma unroll
          for (int e = 0; e < 8; ++e) d[e >> 2][e & 3] = log_decay<RULE>(a, h, c + e, d[e >> 2][e & 3]) * kLog2e;
        }
      *reinterpret_cast<f4 *>(&sG[r * LDG + c]) = d[0], *reinterpret_cast<f4 *>(&sG[r * LDG + c + 4]) = d[1];
    }
  }
  if (tid < C) {
    float b = 0.f;
    if constexpr (DELTA)
      if (tid < n)
        b = sigmoid_f(sum_at(a.y, (size_t)a.T * a.y.NP, (size_t)(sp.t0 + t0 + tid) * a.y.NP + a.col_beta + h));
    sbeta[tid] = b;
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

  if constexpr (!DELTA) {  // the values as they are
    for (int c = tid; c < C * (a.vs / 8); c += 256) {
      const int r = c / (a.vs / 8), col = c % (a.vs / 8) * 8;
      f4 v[2];
      v[0] = v[1] = f4{0.f, 0.f, 0.f, 0.f};
      if (r < n) {
        if (col < a.vg) project8(a, sp, bank, t0 + r, 2 * a.G * a.dg + h * a.vg + col, true, v);
        if constexpr (RULE == kMemoryNormed)
#pragma unroll
          for (int e = 0; e < 8; ++e)
            if (col + e == a.vdim) v[e >> 2][e & 3] = 1.f;
      }
      *reinterpret_cast<uint4 *>((uint16_t *)w.u + (id * C + r) * a.vs + col) = pack8_bf16(v[0], v[1]);
    }
  } else {
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
      for (int i = tid; i < C * VW / 8; i += 256) {
        const int r = i / (VW / 8), c = i % (VW / 8) * 8;
        f4 v[2];
        v[0] = v[1] = f4{0.f, 0.f, 0.f, 0.f};
        if (r < n && c0 + c < a.vg) project8(a, sp, bank, t0 + r, 2 * a.G * a.dg + h * a.vg + c0 + c, true, v);
        *reinterpret_cast<uint4 *>(&sV[r * LDV + c]) = pack8_bf16(v[0], v[1]);
      }
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
        *reinterpret_cast<f4 *>((float *)w.u + (id * C + ri) * a.vs + c0 + ct * 16 + 4 * g) = x;
      }
    }
  }
}

// The pass over the chunks: a workgroup per (VS state columns, head, span).  Wave w: rows
// 16 w .. of u and o, and of the state 16 columns and an even share of the rows, in
// registers (lane: 4 rows of one column); the state goes to LDS once a chunk as the
// operand [column][row], u as rows.  What the next chunk needs is fetched a chunk ahead.
template <bool DELTA, int KS, int VS>
__global__ __launch_bounds__(256, KS * VS <= (DELTA ? 64 : 128) ? 2 : 1) void memory_scan_kernel(const char *__restrict__ blob, int off_spans,
                                                                           Memory a, MemoryScratch w, int limit) {
  constexpr int DK = KS * 32, LDK = DK + 8, LDU = VS + 8;
  constexpr int VT = VS / 16, WD = 4 / VT, ND = (2 * KS + WD - 1) / WD;
  __shared__ __attribute__((aligned(16))) uint16_t sHi[VS * LDK], sLo[VS * LDK], sU[C * LDU], sUl[DELTA ? C * LDU : 8];
  const PagedSpan sp = reinterpret_cast<const PagedSpan *>(blob + off_spans)[blockIdx.z];
  if (sp.n <= limit) return;
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, l15 = lane & 15;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.y, c0 = blockIdx.x * VS, vw = min(VS, a.vs - c0);
  const int ri = wave * 16 + l15, vcol = wave % VT * 16 + l15, d0 = wave / VT * ND;
  const size_t id0 = ((size_t)(sp.t0 / C) + blockIdx.z) * a.H + h;

  bf8 fq[KS], fw[DELTA ? KS : 1], fp[2], fk[ND][2];
  f4 fu[VT], fl[ND];
  uint2 fv[VT];
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
      const size_t at = (id * C + ri) * a.vs + c0 + min(vt * 16, vw - 16) + 4 * g;
      if constexpr (DELTA) fu[vt] = *reinterpret_cast<const f4 *>((const float *)w.u + at);
      else fv[vt] = *reinterpret_cast<const uint2 *>((const uint16_t *)w.u + at);
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
        *reinterpret_cast<uint2 *>(&sU[at]) = fv[vt];
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

// norm and gate of a long span's outputs: sixteen lanes a (token, head)
template <MemoryRule RULE>
__global__ __launch_bounds__(256) void memory_out_kernel(const char *__restrict__ blob, Memory a, MemoryScratch w,
                                                         int limit) {
  const int l15 = threadIdx.x & 15;
  const long id = blockIdx.x * 16L + (threadIdx.x >> 4);
  const int t = (int)min(id / a.H, (long)a.T - 1), h = (int)(id % a.H);
  const PagedToken tk = reinterpret_cast<const PagedToken *>(blob + a.off_tokens)[t];
  const bool mine = id < (long)a.T * a.H && tk.back + tk.ahead + 1 > limit;
  const float *o = w.o + ((size_t)t * a.H + h) * a.vs;
  float f = 1.f, ss = 0.f;
  if (mine) {
    if constexpr (RULE == kMemoryNormed)
      f = __fdiv_rn(1.0f, fmaxf(fabsf(o[a.vdim]), expf(-w.gates[((size_t)t * a.H + h) * 3 + 2])) + 1e-6f);
    for (int c = l15 * 4; c < a.vdim; c += 64) {
      const f4 v = *reinterpret_cast<const f4 *>(o + c) * f;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (c + e < a.vdim) ss = fmaf(v[e], v[e], ss);
    }
  }
#pragma unroll
  for (int k = 1; k < 16; k <<= 1) ss += __shfl_xor(ss, k);
  if (!mine) return;
  const float r = f * inv_rms(ss, a.vdim, a.eps);
  const bool second = a.gate.r > 0;
  const Partials &gp = second ? a.z : a.y;
  const size_t gat = (size_t)t * gp.NP + (second ? a.gate.zcol : a.col_gate) + h * a.vg;
  for (int c = l15 * 8; c < a.vg; c += 128) {
    f4 v[2], gt[2];
    sum8(gp, (size_t)a.T * gp.NP, gat + c, gt);
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      v[j] = *reinterpret_cast<const f4 *>(o + c + 4 * j);
      const f4 wv = *reinterpret_cast<const f4 *>(a.norm + (a.norm_heads ? h * a.vg : 0) + c + 4 * j);
#pragma unroll
      for (int e = 0; e < 4; ++e)
        v[j][e] = c + 4 * j + e < a.vdim ? v[j][e] * r * wv[e] * (a.gate_silu ? silu_f(gt[j][e]) : sigmoid_f(gt[j][e])) : 0.f;
    }
    *reinterpret_cast<uint4 *>((uint16_t *)a.out + act_packed_off(t, a.out_col + h * a.vg + c, a.ldo)) = pack8_bf16(v[0], v[1]);
  }
}

template <MemoryRule RULE>
hipError_t run_chunks(const char *blob, int off_spans, int num_spans, const Memory &a, const MemoryScratch &w,
                      int limit, hipStream_t s) {
  constexpr bool DELTA = RULE == kMemoryDelta;
  const int chunks = (a.T + C - 1) / C;  // (of the longest span there can be)
  if (RULE == kMemoryNormed)
    hipLaunchKernelGGL(memory_gates_kernel, dim3(a.H, num_spans), dim3(256), 0, s, blob, off_spans, a, w, limit);
  // narrow workgroups where the spans and heads alone do not fill the chip
  const bool wide = (long)a.H * num_spans * (a.vs / 32) >= 256;
#define FFMI_MS(KS, VS)                                                                                              \
  hipLaunchKernelGGL((memory_scan_kernel<DELTA, KS, VS>), dim3((a.vs + VS - 1) / VS, a.H, num_spans), dim3(256), 0, s, \
                     blob, off_spans, a, w, limit)
#define FFMI_MC(KS)                                                                                               \
  do {                                                                                                            \
    hipLaunchKernelGGL((memory_chunk_kernel<RULE, KS>), dim3(chunks, a.H, num_spans), dim3(256), 0, s, blob,       \
                       off_spans, a, w, limit);                                                                   \
    if (wide) FFMI_MS(KS, 32);                                                                                    \
    else FFMI_MS(KS, 16);                                                                                         \
  } while (0)
  switch (memory_chunk_width(a.dg)) {
    case 32: FFMI_MC(1); break;
    case 64: FFMI_MC(2); break;
    case 128: FFMI_MC(4); break;
    default: FFMI_MC(8); break;
  }
#undef FFMI_MC
#undef FFMI_MS
  hipLaunchKernelGGL(memory_out_kernel<RULE>, dim3((unsigned)(((long)a.T * a.H + 15) / 16)), dim3(256), 0, s, blob, a,
                     w, limit);
  return hipGetLastError();
}

}  // namespace

hipError_t launch_memory_chunks(const char *blob, int off_spans, int num_spans, const Memory &a,
                                const MemoryScratch &w, int limit, hipStream_t s) {
  if (num_spans <= 0) return hipSuccess;
  if (a.H < 1 || a.G < 1 || a.H % a.G || a.dg % 32 || a.vg % 32 || a.dg > kMemoryMaxChunkDim || a.dim > a.dg ||
      a.vdim > a.vg || a.vs != memory_state_columns(a.rule, a.vdim) || a.y.S < 1 || a.y.NP % 4 || a.col % 4 ||
      a.col_gate % 4 || a.decay.zcol % 4 || a.gate.zcol % 4 || limit < a.taps || a.ldo % 32 || a.out_col % 32 ||
      (a.taps > 0 && !a.conv) || (a.taps > 1 && !a.carry) || (a.rule != kMemoryNormed && (a.z.S < 1 || a.z.NP % 4)) ||
      !w.qg || !w.kd || !w.p || !w.u || !w.last || !w.o || (a.rule == kMemoryDelta && !w.w) ||
      (a.rule == kMemoryNormed && !w.gates))
    return hipErrorInvalidValue;
  if (a.rule == kMemoryGated) return run_chunks<kMemoryGated>(blob, off_spans, num_spans, a, w, limit, s);
  if (a.rule == kMemoryDelta) return run_chunks<kMemoryDelta>(blob, off_spans, num_spans, a, w, limit, s);
  return run_chunks<kMemoryNormed>(blob, off_spans, num_spans, a, w, limit, s);
}

}  // namespace ffmi
