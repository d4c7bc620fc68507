// lightning.hip -- linear attention with a fixed decay per head (lightning.h).
#include "lightning.h"

#include <algorithm>

#include "device_util.h"

namespace ffmi {

typedef short s4 __attribute__((ext_vector_type(4)));
typedef uint32_t u4 __attribute__((ext_vector_type(4)));

// ---------------------------------------------------------------------------
// token by token: a workgroup per (32 value columns, head, span), the state in
// registers: thread = (row ri of every 32 rows, 4 columns)
// ---------------------------------------------------------------------------
template <int P>
__global__ __launch_bounds__(256) void lightning_recurrent_kernel(const char *__restrict__ blob,
                                                                  int off_spans, Lightning a,
                                                                  int limit) {
  __shared__ float sq[2][P * 32], sk[2][P * 32], sv[2][32], red[2][4][32];
  const PagedSpan sp = reinterpret_cast<const PagedSpan *>(blob + off_spans)[blockIdx.z];
  if (sp.n > limit) return;
  const int tid = threadIdx.x, h = blockIdx.y, c0 = blockIdx.x * 32;
  const int cl = (tid & 7) * 4, ri = tid >> 3;
  float *S = a.state + (((size_t)sp.slot * a.H + h) * a.dg) * a.vg + c0 + cl;
  const float decay = a.powers[(size_t)h * (kLightningChunk + 1) + 1];
  f4 st[P];
#pragma unroll
  for (int p = 0; p < P; ++p) {
    const int row = p * 32 + ri;
    st[p] = f4{0.f, 0.f, 0.f, 0.f};
    if (sp.pos0 > 0 && row < a.dg) st[p] = *reinterpret_cast<const f4 *>(S + (size_t)row * a.vg);
  }
  const size_t slab = (size_t)a.T * a.y.NP;
  const size_t colk = (size_t)a.H * a.dg, colv = 2 * colk;
  auto load = [&](int t, int b) {
    const size_t row = (size_t)(sp.t0 + t) * a.y.NP;
    for (int i = tid; i < 2 * a.dg + 32; i += 256) {
      if (i < a.dg) sq[b][i] = silu_f(sum_at(a.y, slab, row + (size_t)h * a.dg + i));
      else if (i < 2 * a.dg) sk[b][i - a.dg] = silu_f(sum_at(a.y, slab, row + colk + (size_t)h * a.dg + i - a.dg));
      else sv[b][i - 2 * a.dg] = silu_f(sum_at(a.y, slab, row + colv + (size_t)h * a.vg + c0 + i - 2 * a.dg));
    }
  };
  load(0, 0);
  for (int t = 0; t < sp.n; ++t) {
    const int b = t & 1;
    __syncthreads();
    const f4 v = *reinterpret_cast<const f4 *>(&sv[b][cl]);
    f4 o = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int p = 0; p < P; ++p) {
      const int row = p * 32 + ri;
      if (row >= a.dg) continue;
      const float k = sk[b][row], q = sq[b][row];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        st[p][e] = fmaf(decay, st[p][e], k * v[e]);
        o[e] = fmaf(q, st[p][e], o[e]);
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      o[e] += __shfl_xor(o[e], 8);
      o[e] += __shfl_xor(o[e], 16);
      o[e] += __shfl_xor(o[e], 32);
    }
    if ((tid & 63) < 8) *reinterpret_cast<f4 *>(&red[b][tid >> 6][cl]) = o;
    if (t + 1 < sp.n) load(t + 1, b ^ 1);
    __syncthreads();
    if (tid < 32)
      a.o[(size_t)(sp.t0 + t) * a.H * a.vg + (size_t)h * a.vg + c0 + tid] =
          red[b][0][tid] + red[b][1][tid] + red[b][2][tid] + red[b][3][tid];
  }
#pragma unroll
  for (int p = 0; p < P; ++p) {
    const int row = p * 32 + ri;
    if (row < a.dg) *reinterpret_cast<f4 *>(S + (size_t)row * a.vg) = st[p];
  }
}

static bool bad_shape(const Lightning &a, int max_dim) {
  return a.H < 1 || a.dg % 32 || a.vg % 32 || a.dg < 32 || a.vg < 32 || a.dg > max_dim || a.y.S < 1 ||
         a.y.NP < 2 * a.H * (a.dg + a.vg);
}

hipError_t launch_lightning_recurrent(const char *blob, int off_spans, int num_spans,
                                      const Lightning &a, int limit, hipStream_t s) {
  if (num_spans <= 0) return hipSuccess;
  if (bad_shape(a, kLightningMaxDim)) return hipErrorInvalidValue;
  const dim3 grid(a.vg / 32, a.H, num_spans);
#define FFMI_LR(P)                                                                                 \
  hipLaunchKernelGGL((lightning_recurrent_kernel<P>), grid, dim3(256), 0, s, blob, off_spans, a, limit)
  if (a.dg <= 32) FFMI_LR(1);
  else if (a.dg <= 64) FFMI_LR(2);
  else if (a.dg <= 128) FFMI_LR(4);
  else if (a.dg <= 256) FFMI_LR(8);
  else FFMI_LR(16);
#undef FFMI_LR
  return hipGetLastError();
}

// ---------------------------------------------------------------------------
// chunks
// ---------------------------------------------------------------------------
// silu of the q | k | v columns, 8 a thread
__global__ __launch_bounds__(256) void lightning_qkv_kernel(Lightning a, int cols) {
  const int n8 = cols / 8;
  const long id = blockIdx.x * 256L + threadIdx.x;
  if (id >= (long)a.T * n8) return;
  const int t = (int)(id / n8), c = (int)(id % n8) * 8;
  const float *p = a.y.p + (size_t)t * a.y.NP + c;
  f4 lo = *reinterpret_cast<const f4 *>(p), hi = *reinterpret_cast<const f4 *>(p + 4);
  for (int s = 1; s < a.y.S; ++s) {
    const float *ps = p + (size_t)s * a.T * a.y.NP;
    lo += *reinterpret_cast<const f4 *>(ps), hi += *reinterpret_cast<const f4 *>(ps + 4);
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) lo[e] = silu_f(lo[e]), hi[e] = silu_f(hi[e]);
  *reinterpret_cast<uint4 *>(a.qkv + (size_t)t * cols + c) = pack8_bf16(lo, hi);
}

// operand of 8 k-values from row-major LDS rows: column c0 + (lane & 15), rows
// kb * 32 + {4g .. 4g + 3, 16 + 4g ..}
template <int LD>
__device__ __forceinline__ bf8 read_columns(const uint16_t *tile, int kb, int c0) {
  const int lane = threadIdx.x & 63, g = lane >> 4, l15 = lane & 15;
  const uint16_t *p = tile + (kb * 32 + 4 * g + (l15 >> 2)) * LD + c0 + 4 * (l15 & 3);
  const s4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4 *)(p));
  const s4 hi =
      __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s4 *)(p + 16 * LD));
  return __builtin_bit_cast(bf8, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
}

// A workgroup per (VS value columns, head, span).  Per chunk of 64 tokens
//   O^T = S_prev^T Q^T, row i times d^(i + 1),  + V^T . P^T with
//   P = (q_i . k_j) d^(i - j) for j <= i;
//   S   = d^n S_prev + K^T . (v_j d^(n - 1 - j))
// Wave w: rows 16 w .. of the outputs, and of the state 16 value columns and
// an even share of the rows.  Its part of the state stays in its registers
// (lane: 4 rows of one column) and goes to LDS once a chunk as the operand
// [column][row] of every wave's outputs.
template <int KS, int VS>
__global__ __launch_bounds__(256, KS <= 4 || VS == 16 ? 2 : 1) void lightning_chunk_kernel(const char *__restrict__ blob,
                                                              int off_spans, Lightning a, int limit) {
  constexpr int DK = KS * 32, LDK = DK + 8, LDV = VS + 8, C = kLightningChunk;
  constexpr int VT = VS / 16, WD = 4 / VT;        // value tiles; waves that share one
  constexpr int ND = (2 * KS + WD - 1) / WD;      // a wave's row tiles of the state
  constexpr int NV = (C * VS / 8 + 255) / 256;    // 16-byte chunks of V per thread
  __shared__ __attribute__((aligned(16))) uint16_t sK[C * LDK], sV[C * LDV], sHi[VS * LDK], sLo[VS * LDK];
  __shared__ float pw[C + 1];
  const PagedSpan sp = reinterpret_cast<const PagedSpan *>(blob + off_spans)[blockIdx.z];
  if (sp.n <= limit) return;
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, l15 = lane & 15;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.y, c0 = blockIdx.x * VS, cols = a.H * (2 * a.dg + a.vg);
  const uint16_t *Q = a.qkv + (size_t)sp.t0 * cols + (size_t)h * a.dg;
  const uint16_t *K = Q + (size_t)a.H * a.dg;
  const uint16_t *V = a.qkv + (size_t)sp.t0 * cols + (size_t)2 * a.H * a.dg + (size_t)h * a.vg + c0;
  if (tid <= C) pw[tid] = a.powers[(size_t)h * (C + 1) + tid];
  const int vw = min(VS, a.vg - c0);  // value columns of this workgroup
  const int i = wave * 16 + l15;      // this lane's row of the chunk

  const u4 zero = {0, 0, 0, 0};
  u4 pk[KS], pv[NV], pq[KS];
  auto fetch = [&](int t0) {  // rows past the span and columns past the widths: zeros
#pragma unroll
    for (int j = 0; j < KS; ++j) {
      const int ch = tid + j * 256, r = ch / (DK / 8), c = ch % (DK / 8) * 8;
      pk[j] = zero;
      if (t0 + r < sp.n && c < a.dg) pk[j] = *reinterpret_cast<const u4 *>(K + (size_t)(t0 + r) * cols + c);
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int ch = tid + j * 256, r = ch / (VS / 8), c = ch % (VS / 8) * 8;
      pv[j] = zero;
      if (r < C && t0 + r < sp.n && c < vw)
        pv[j] = *reinterpret_cast<const u4 *>(V + (size_t)(t0 + r) * cols + c);
    }
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      pq[ks] = zero;
      if (t0 + i < sp.n && ks * 32 < a.dg)
        pq[ks] = *reinterpret_cast<const u4 *>(Q + (size_t)(t0 + i) * cols + ks * 32 + 8 * g);
    }
  };
  auto stage = [&]() {
#pragma unroll
    for (int j = 0; j < KS; ++j) {
      const int ch = tid + j * 256;
      *reinterpret_cast<u4 *>(&sK[(ch / (DK / 8)) * LDK + ch % (DK / 8) * 8]) = pk[j];
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int ch = tid + j * 256, r = ch / (VS / 8);
      if (r < C) *reinterpret_cast<u4 *>(&sV[r * LDV + ch % (VS / 8) * 8]) = pv[j];
    }
  };
  fetch(0);
  // the state: rows (d0 + dt) * 16 + 4g + e, column vcol
  f4 st[ND];
  const int vcol = wave % VT * 16 + l15, d0 = wave / VT * ND;
  float *S = a.state + (((size_t)sp.slot * a.H + h) * a.dg) * a.vg + c0 + vcol;
#pragma unroll
  for (int dt = 0; dt < ND; ++dt) {
    st[dt] = f4{0.f, 0.f, 0.f, 0.f};
    if (sp.pos0 > 0 && (d0 + dt) * 16 < a.dg && vcol < vw)
#pragma unroll
      for (int e = 0; e < 4; ++e) st[dt][e] = S[(size_t)((d0 + dt) * 16 + 4 * g + e) * a.vg];
  }
  auto publish = [&]() {
#pragma unroll
    for (int dt = 0; dt < ND; ++dt) {
      if (2 * KS % WD && d0 + dt >= 2 * KS) continue;
      __bf16 hi[4], lo[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) split2(st[dt][e], hi[e], lo[e]);
      const int at = vcol * LDK + (d0 + dt) * 16 + 4 * g;
      auto two = [](const __bf16 *v) {
        return make_uint2(__builtin_bit_cast(uint16_t, v[0]) | ((uint32_t)__builtin_bit_cast(uint16_t, v[1]) << 16),
                          __builtin_bit_cast(uint16_t, v[2]) | ((uint32_t)__builtin_bit_cast(uint16_t, v[3]) << 16));
      };
      *reinterpret_cast<uint2 *>(&sHi[at]) = two(hi);
      *reinterpret_cast<uint2 *>(&sLo[at]) = two(lo);
    }
  };
  publish();
  __syncthreads();  // (pw)
  // this lane's decays: of its weights (key <= row), of its row, of its values
  const auto key_of = [&](int kb, int e) { return kb * 32 + 4 * g + (e & 3) + 16 * (e >> 2); };
  float fp[2][8], fv[2][8];
#pragma unroll
  for (int kb = 0; kb < 2; ++kb)
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int key = key_of(kb, e);
      fp[kb][e] = key <= i ? pw[max(i - key, 0)] : 0.f;
      fv[kb][e] = pw[C - 1 - key];
    }
  const float fi = pw[i + 1];
  for (int t0 = 0; t0 < sp.n; t0 += C) {
    const int n = min(C, sp.n - t0);
    if (n < C)  // (rows past the span are zeros)
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int e = 0; e < 8; ++e) fv[kb][e] = pw[max(n - 1 - key_of(kb, e), 0)];
    stage();
    bf8 q[KS];
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) q[ks] = __builtin_bit_cast(bf8, pq[ks]);
    __syncthreads();
    if (t0 + C < sp.n) fetch(t0 + C);
    // from the state before the chunk: value and remainder, a chain each
    f4 o[VT], olo[VT];
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) o[vt] = olo[vt] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) {
        const int at = (vt * 16 + l15) * LDK + ks * 32 + 8 * g;
        o[vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf8 *>(&sHi[at]), q[ks],
                                                        o[vt], 0, 0, 0);
        olo[vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf8 *>(&sLo[at]), q[ks],
                                                          olo[vt], 0, 0, 0);
      }
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) o[vt] = (o[vt] + olo[vt]) * fi;
    // within the chunk: keys of 32 at a time
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      if (kb * 32 > wave * 16 + 15) continue;  // (all after this wave's rows)
      bf8 ph, plo;
      f4 s[2];
      s[0] = s[1] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks)
#pragma unroll
        for (int j = 0; j < 2; ++j)
          s[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              *reinterpret_cast<const bf8 *>(&sK[(kb * 32 + j * 16 + l15) * LDK + ks * 32 + 8 * g]), q[ks],
              s[j], 0, 0, 0);
#pragma unroll
      for (int j = 0; j < 2; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          __bf16 hi, lo;
          split2(s[j][e] * fp[kb][j * 4 + e], hi, lo);
          ph[j * 4 + e] = hi, plo[j * 4 + e] = lo;
        }
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) {
        const bf8 v = read_columns<LDV>(sV, kb, vt * 16);
        o[vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, ph, o[vt], 0, 0, 0);
        o[vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, plo, o[vt], 0, 0, 0);
      }
    }
    // the state after the chunk
    const float dn = pw[n];
#pragma unroll
    for (int dt = 0; dt < ND; ++dt) st[dt] *= dn;
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      const bf8 v = read_columns<LDV>(sV, kb, wave % VT * 16);
      bf8 vh, vl;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        __bf16 hi, lo;
        split2((float)v[e] * fv[kb][e], hi, lo);
        vh[e] = hi, vl[e] = lo;
      }
#pragma unroll
      for (int dt = 0; dt < ND; ++dt) {
        if (2 * KS % WD && d0 + dt >= 2 * KS) continue;
        const bf8 k = read_columns<LDK>(sK, kb, (d0 + dt) * 16);
        st[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, vh, st[dt], 0, 0, 0);
        st[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, vl, st[dt], 0, 0, 0);
      }
    }
    if (i < n) {
      float *dst = a.o + (size_t)(sp.t0 + t0 + i) * a.H * a.vg + (size_t)h * a.vg + c0 + 4 * g;
#pragma unroll
      for (int vt = 0; vt < VT; ++vt)
        if (vt * 16 < vw) *reinterpret_cast<f4 *>(dst + vt * 16) = o[vt];
    }
    __syncthreads();
    if (t0 + C < sp.n) publish();
  }
#pragma unroll
  for (int dt = 0; dt < ND; ++dt)
    if ((d0 + dt) * 16 < a.dg && vcol < vw)
#pragma unroll
      for (int e = 0; e < 4; ++e) S[(size_t)((d0 + dt) * 16 + 4 * g + e) * a.vg] = st[dt][e];
}

hipError_t launch_lightning_chunks(const char *blob, int off_spans, int num_spans, const Lightning &a,
                                   int limit, hipStream_t s) {
  if (num_spans <= 0) return hipSuccess;
  if (bad_shape(a, kLightningMaxChunkDim) || !a.qkv) return hipErrorInvalidValue;
  const int cols = a.H * (2 * a.dg + a.vg);
  const long n = (long)a.T * (cols / 8);
  hipLaunchKernelGGL(lightning_qkv_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, s, a, cols);
  // narrow workgroups where the spans and heads alone do not fill the chip
  const long wide = (long)a.H * num_spans * ((a.vg + 63) / 64);
#define FFMI_LC2(KS, VS)                                                                                  \
  hipLaunchKernelGGL((lightning_chunk_kernel<KS, VS>), dim3((a.vg + VS - 1) / VS, a.H, num_spans), dim3(256), \
                     0, s, blob, off_spans, a, limit)
#define FFMI_LC(KS)                        \
  do {                                     \
    if (wide <= 128) FFMI_LC2(KS, 16);     \
    else if (wide <= 256) FFMI_LC2(KS, 32); \
    else FFMI_LC2(KS, 64);                 \
  } while (0)
  if (a.dg <= 32) FFMI_LC(1);
  else if (a.dg <= 64) FFMI_LC(2);
  else if (a.dg <= 128) FFMI_LC(4);
  else FFMI_LC(8);
#undef FFMI_LC
#undef FFMI_LC2
  return hipGetLastError();
}

// ---------------------------------------------------------------------------
// norm over all heads, gate
// ---------------------------------------------------------------------------
__global__ __launch_bounds__(256) void gated_norm_kernel(const float *__restrict__ o, Partials y,
                                                         int gate_col, const float *__restrict__ w,
                                                         uint16_t *__restrict__ hb,
                                                         float *__restrict__ hf, int H, int n,
                                                         float eps) {
  __shared__ float sh[4];
  const int t = blockIdx.x, T = gridDim.x;
  const float *row = o + (size_t)t * H;
  float ss = 0.f;
  for (int c = threadIdx.x; c < H / 4; c += 256) {
    const f4 v = *reinterpret_cast<const f4 *>(row + c * 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) ss = fmaf(v[e], v[e], ss);
  }
  const float r = inv_rms(row_sum<256>(ss, sh), n, eps);
  for (int c = threadIdx.x; c < H / 8; c += 256) {
    f4 v[2];
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      const int at = c * 8 + 4 * k;
      const float *gp = y.p + (size_t)t * y.NP + gate_col + at;
      f4 gt = *reinterpret_cast<const f4 *>(gp);
      for (int s = 1; s < y.S; ++s) gt += *reinterpret_cast<const f4 *>(gp + (size_t)s * T * y.NP);
      v[k] = *reinterpret_cast<const f4 *>(row + at);
      const f4 wv = *reinterpret_cast<const f4 *>(w + at);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[k][e] = v[k][e] * r * wv[e] * sigmoid_f(gt[e]);
      if (hf) *reinterpret_cast<f4 *>(hf + (size_t)t * H + at) = v[k];
    }
    if (hb) *reinterpret_cast<uint4 *>(hb + act_packed_off(t, c * 8, H)) = pack8_bf16(v[0], v[1]);
  }
}
hipError_t launch_gated_norm(const float *o, const Partials &y, int gate_col, const float *w,
                             uint16_t *hb, float *hf, int T, int H, int n, float eps, hipStream_t s) {
  if (T <= 0) return hipSuccess;
  if (H % 32 || gate_col % 4 || y.S < 1) return hipErrorInvalidValue;
  hipLaunchKernelGGL(gated_norm_kernel, dim3(T), dim3(256), 0, s, o, y, gate_col, w, hb, hf, H, n, eps);
  return hipGetLastError();
}

}  // namespace ffmi
