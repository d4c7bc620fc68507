// paged_attn_kernels.h -- attention over paged keys and values (paged_attn.h).
// Included by paged_attn.hip (kind kBias) and rotary_attn.hip (kind kRotary), one
// translation unit per kind.
#pragma once
#include <algorithm>

#include "device_util.h"
#include "paged_attn.h"

namespace ffmi {

typedef uint32_t u4 __attribute__((ext_vector_type(4)));
typedef float f2 __attribute__((ext_vector_type(2)));

// What the scores and the queries, keys and values are made of:
//   kBias    norm and temperature per head, mixed values; scores + bias by distance
//   kRotary  optional norm over whole rows, rotation; soft-capped scores, window,
//            sink, values that turn with their position
enum AttnKind { kBias = 0, kRotary = 1 };

// ---------------------------------------------------------------------------
// queries, keys, values: one wave per (tokens, head)
// ---------------------------------------------------------------------------
// column n of a row of deferred sums; several slabs: their loads together
__device__ __forceinline__ float slab_sum(const Partials &y, size_t slab, size_t at) {
  float v = y.p[at];
  if (y.S > 1) {
    float p[7];
#pragma unroll
    for (int s = 1; s < 8; ++s) p[s - 1] = y.p[at + (size_t)min(s, y.S - 1) * slab];
#pragma unroll
    for (int s = 1; s < 8; ++s)
      if (s < y.S) v += p[s - 1];
  }
  return v;
}

__device__ __forceinline__ void store4(uint16_t *p, float a, float b, float c, float d) {
  *reinterpret_cast<uint2 *>(p) =
      make_uint2(f2bf(a) | ((uint32_t)f2bf(b) << 16), f2bf(c) | ((uint32_t)f2bf(d) << 16));
}
__device__ __forceinline__ void store4(float *p, float a, float b, float c, float d) {
  *reinterpret_cast<f4 *>(p) = f4{a, b, c, d};
}

__device__ __forceinline__ f2 slab_sum2(const Partials &y, size_t slab, size_t at) {
  f2 v = *reinterpret_cast<const f2 *>(y.p + at);
  if (y.S > 1) {
    f2 p[7];
#pragma unroll
    for (int s = 1; s < 8; ++s)
      p[s - 1] = *reinterpret_cast<const f2 *>(y.p + at + (size_t)min(s, y.S - 1) * slab);
#pragma unroll
    for (int s = 1; s < 8; ++s)
      if (s < y.S) v[0] += p[s - 1][0], v[1] += p[s - 1][1];
  }
  return v;
}
__device__ __forceinline__ void store2(uint16_t *p, f2 v) {
  *reinterpret_cast<uint32_t *>(p) = f2bf(v[0]) | ((uint32_t)f2bf(v[1]) << 16);
}
__device__ __forceinline__ void store2(float *p, f2 v) { *reinterpret_cast<f2 *>(p) = v; }

// One head of one token across a wave: a lane holds NE columns in neighbouring
// pairs (NE == 1: one column).  Heads in the order of the columns: q, k, v.
template <int NE>
__device__ __forceinline__ int head_column(int i) {
  const int lane = threadIdx.x & 63;
  return NE == 1 ? lane : (i >> 1) * 128 + lane * 2 + (i & 1);
}
__device__ __forceinline__ int head_width(const AttnPrep &a, int hd) {
  return hd >= a.H + a.G ? a.vg : a.dg;
}
__device__ __forceinline__ int head_start(const AttnPrep &a, int hd) {
  return hd >= a.H + a.G ? (a.H + a.G) * a.dg + (hd - a.H - a.G) * a.vg : hd * a.dg;
}
template <int NE>
__device__ __forceinline__ void load_bias(const AttnPrep &a, int hd, float (&b)[NE]) {
#pragma unroll
  for (int i = 0; i < NE; ++i) b[i] = 0.f;
  if (!a.bias) return;
  const float *p = a.bias + head_start(a, hd);
  if constexpr (NE == 1) {
    const int c = head_column<NE>(0);
    if (c < head_width(a, hd)) b[0] = p[c];
  } else {
#pragma unroll
    for (int i = 0; i < NE; i += 2) {
      const int c = head_column<NE>(i);
      if (c >= head_width(a, hd)) continue;
      const f2 v = *reinterpret_cast<const f2 *>(p + c);
      b[i] = v[0], b[i + 1] = v[1];
    }
  }
}
// its product, with the bias
template <int NE>
__device__ __forceinline__ void load_head(const AttnPrep &a, int T, int t, int hd, const float (&b)[NE],
                                          float (&v)[NE]) {
  const int wd = head_width(a, hd);
  const size_t slab = (size_t)T * a.y.NP, row = (size_t)t * a.y.NP + head_start(a, hd);
  if constexpr (NE == 1) {
    const int c = head_column<NE>(0);
    v[0] = 0.f;
    if (c < wd) v[0] = slab_sum(a.y, slab, row + c) + b[0];
  } else {
#pragma unroll
    for (int i = 0; i < NE; i += 2) {
      const int c = head_column<NE>(i);  // (the widths are even)
      v[i] = v[i + 1] = 0.f;
      if (c < wd) {
        const f2 p = slab_sum2(a.y, slab, row + c);
        v[i] = p[0] + b[i], v[i + 1] = p[1] + b[i + 1];
      }
    }
  }
}
// (rotary kind, few rows) The convolution over time of one head's columns: v, a token's
// product, becomes the sum over its taps, and the rows that later steps need go to the
// other bank.  Up to TAPS taps: their weights and the earlier rows are asked for with the
// product (load).
template <int NE>
struct HeadConv {
  static constexpr int TAPS = 4, PAST = TAPS - 1;
  float w[TAPS][NE], x[PAST][NE];  // of the token d back, and its row
  static __device__ __forceinline__ size_t columns(const AttnPrep &a) {
    return (size_t)(a.H + a.G) * a.dg + (size_t)a.G * a.vg;
  }
  static __device__ __forceinline__ const float *bank(const AttnPrep &a, const PagedToken &tk, int other) {
    return a.carry + ((size_t)tk.slot * 2 + (tk.bank ^ other)) * (a.taps - 1) * columns(a);
  }
  // column col d tokens before token t (0: before the sequence)
  static __device__ __forceinline__ float before(const AttnPrep &a, int T, int t, const PagedToken &tk, int d,
                                                 size_t col) {
    if (d > tk.pos) return 0.f;
    if (tk.back >= d) return sum_at(a.y, (size_t)T * a.y.NP, (size_t)(t - d) * a.y.NP + col);
    return bank(a, tk, 0)[(d - tk.back - 1) * columns(a) + col];
  }
  __device__ __forceinline__ void load(const AttnPrep &a, int T, int t, const PagedToken &tk, int hd) {
    const int wd = head_width(a, hd), c0 = head_start(a, hd), past = a.taps - 1;
    if (past > PAST) return;
    const size_t C = columns(a);
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int c = head_column<NE>(i);
#pragma unroll
      for (int d = 0; d <= PAST; ++d) {
        w[d][i] = c < wd && d <= past ? a.conv[(past - d) * C + c0 + c] : 0.f;
        if (d > 0) x[d - 1][i] = c < wd && d <= past ? before(a, T, t, tk, d, c0 + c) : 0.f;
      }
    }
  }
  __device__ __forceinline__ void apply(const AttnPrep &a, int T, int t, const PagedToken &tk, int hd,
                                        float (&v)[NE]) {
    const int wd = head_width(a, hd), c0 = head_start(a, hd), past = a.taps - 1;
    const size_t C = columns(a);
    float *now = const_cast<float *>(bank(a, tk, 1));
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int c = head_column<NE>(i);
      if (c >= wd) continue;
      const size_t col = c0 + c;
      const float u = v[i];
      if (tk.ahead < past) now[tk.ahead * C + col] = u;
      if (past <= PAST) {
        if (tk.back == 0)  // (a short portion: earlier rows move on)
#pragma unroll
          for (int d = 1; d <= PAST; ++d)
            if (tk.ahead + d < past) now[(tk.ahead + d) * C + col] = x[d - 1][i];
        float sum = u * w[0][i];
#pragma unroll
        for (int d = 1; d <= PAST; ++d) sum = fmaf(x[d - 1][i], w[d][i], sum);
        v[i] = sum;
      } else {
        if (tk.back == 0)
          for (int d = 1; tk.ahead + d < past; ++d) now[(tk.ahead + d) * C + col] = before(a, T, t, tk, d, col);
        float sum = u * a.conv[past * C + col];
        for (int d = 1; d <= past; ++d) sum = fmaf(before(a, T, t, tk, d, col), a.conv[(past - d) * C + col], sum);
        v[i] = sum;
      }
    }
  }
};
// values: mixed with, or kept as, the first mixing layer's (lam: *a.vmix)
template <int NE>
__device__ __forceinline__ void mix_head(const AttnPrep &a, int t, int g, float lam, float (&v)[NE]) {
  if (!a.first) return;
  float *first = a.first + ((size_t)t * a.G + g) * a.vg;
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int c = head_column<NE>(i);
    if (c >= a.vg) continue;
    if (a.vmix) v[i] = (1.0f - lam) * v[i] + lam * first[c];
    else first[c] = v[i];
  }
}
// queries and keys: norm, query temperature
template <int NE>
__device__ __forceinline__ void norm_head(const AttnPrep &a, bool isq, int pos, float (&v)[NE]) {
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NE; ++i) ss = fmaf(v[i], v[i], ss);
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) ss += __shfl_xor(ss, o);
  float r = inv_rms(ss, a.dim, a.eps);
  if (isq && a.coef != 0.f) r *= 1.0f + a.coef * logf((float)((pos + 1) / a.every + 1));
  const float *w = a.norms + (isq ? 0 : a.dg);
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int c = head_column<NE>(i);
    v[i] = c < a.dg ? v[i] * r * w[c] : 0.f;
  }
}
// columns 2m, 2m + 1 below `width` turn by pos * freq[m] (in turns)
template <int NE>
__device__ __forceinline__ void rotate_head(const double *freq, int width, float mult, int pos,
                                            float (&v)[NE]) {
  if constexpr (NE == 1) {
    const int c = head_column<NE>(0);
    const float other = __shfl_xor(v[0], 1);
    if (c >= width) return;
    float cs, sn;
    turn_by(pos * freq[c >> 1], cs, sn);
    v[0] = mult * (c & 1 ? v[0] * cs + other * sn : v[0] * cs - other * sn);
  } else {
#pragma unroll
    for (int i = 0; i < NE; i += 2) {
      const int c = head_column<NE>(i);
      if (c >= width) continue;
      float cs, sn;
      turn_by(pos * freq[c >> 1], cs, sn);
      const float x = v[i], y = v[i + 1];
      v[i] = mult * (x * cs - y * sn), v[i + 1] = mult * (y * cs + x * sn);
    }
  }
}
// queries and keys: row norm (r: 1 / rms of the whole row), rotation
template <int NE>
__device__ __forceinline__ void rotary_head(const AttnPrep &a, int hd, int pos, float r, float (&v)[NE]) {
  if (a.norms) {
    const float *w = a.norms + head_start(a, hd);
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int c = head_column<NE>(i);
      if (c < a.dg) v[i] = v[i] * r * w[c];
    }
  }
  if (a.rot > 0) rotate_head<NE>(a.freq, a.rot, a.rot_mult, pos, v);
  if (a.unit) {  // (columns past the head are zero)
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NE; ++i) ss = fmaf(v[i], v[i], ss);
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) ss += __shfl_xor(ss, o);
    const float f = inv_rms(ss, a.dim, a.eps);
#pragma unroll
    for (int i = 0; i < NE; ++i) v[i] *= f;
  }
}
// sums of squares of a token's whole query and key rows: this thread's columns
template <int NTH>
__device__ __forceinline__ void row_squares(const AttnPrep &a, int T, int t, float &sq, float &sk) {
  const size_t slab = (size_t)T * a.y.NP, row = (size_t)t * a.y.NP;
  sq = sk = 0.f;
  for (int c = threadIdx.x * 4; c < (a.H + a.G) * a.dg; c += NTH * 4) {
    f4 v = *reinterpret_cast<const f4 *>(a.y.p + row + c);
    for (int s = 1; s < a.y.S; ++s) v += *reinterpret_cast<const f4 *>(a.y.p + row + c + s * slab);
    if (a.bias) v += *reinterpret_cast<const f4 *>(a.bias + c);
    const float d = fmaf(v[0], v[0], fmaf(v[1], v[1], fmaf(v[2], v[2], v[3] * v[3])));
    if (c < a.H * a.dg) sq += d;
    else sk += d;
  }
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) sq += __shfl_xor(sq, o), sk += __shfl_xor(sk, o);
}
// columns below `width` to dst(column), pairs lying side by side
template <class E, int NE, class D>
__device__ __forceinline__ void store_head(D dst, int width, const float (&v)[NE]) {
  if constexpr (NE == 1) {
    const int c = head_column<NE>(0);
    if (c < width) st_elem((E *)dst(c), v[0]);
  } else {
#pragma unroll
    for (int i = 0; i < NE; i += 2) {
      const int c = head_column<NE>(i);
      if (c < width) store2((E *)dst(c), f2{v[i], v[i + 1]});
    }
  }
}
template <class E, int NE>
__device__ __forceinline__ void store_value(const AttnPrep &a, int crow, int g, const float (&v)[NE]) {
  E *dst = (E *)a.vc + ((size_t)(crow / kPageTokens) * a.G + g) * kPageTokens * a.vp;
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int c = head_column<NE>(i);
    if (c < a.vp) st_elem(dst + val_off(crow % kPageTokens, c, a.vp), v[i]);
  }
}
template <class E, int NE>
__device__ __forceinline__ void store_key(const AttnPrep &a, int crow, int g, const float (&v)[NE]) {
  E *dst = (E *)a.kc + ((size_t)(crow / kPageTokens) * a.G + g) * kPageTokens * a.dp;
  const int key = crow % kPageTokens;
  store_head<E, NE>([&](int c) { return dst + key_off(key, c, a.dp); }, a.dp, v);
}

// A wave takes NT consecutive batch tokens of one head.
template <class E, int NE, int NT>
__global__ __launch_bounds__(256) void attn_prep_kernel(const PagedToken *__restrict__ tok, int T,
                                                        AttnPrep a) {
  const int heads = a.H + 2 * a.G;
  const long id = blockIdx.x * 4L + (threadIdx.x >> 6);
  // (a workgroup's waves side by side in the sequence: the cache lines that
  // they share are written on one CU)
  const int nt = (T + NT - 1) / NT, hd = (int)(id / nt), t0 = (int)(id % nt) * NT;
  if (hd >= heads) return;
  const bool isv = hd >= a.H + a.G, isq = hd < a.H;
  const int g = isq ? 0 : (hd - a.H) % a.G;
  PagedToken tk[NT];
  float v[NT][NE], bias[NE];
  const float lam = isv && a.vmix ? *a.vmix : 0.f;
  load_bias<NE>(a, hd, bias);
#pragma unroll
  for (int k = 0; k < NT; ++k) tk[k] = tok[min(t0 + k, T - 1)];
#pragma unroll
  for (int k = 0; k < NT; ++k) load_head<NE>(a, T, min(t0 + k, T - 1), hd, bias, v[k]);
  if (isv) {
#pragma unroll
    for (int k = 0; k < NT; ++k)
      if (t0 + k < T) mix_head<NE>(a, t0 + k, g, lam, v[k]);
    // four tokens in one aligned run of a page: their values lie side by side
    bool run = NT == 4 && t0 + NT <= T && tk[0].row % 4 == 0;
#pragma unroll
    for (int k = 1; k < NT; ++k) run = run && tk[k].row == tk[0].row + k;
    if (!run) {
#pragma unroll
      for (int k = 0; k < NT; ++k)
        if (t0 + k < T) store_value<E, NE>(a, tk[k].row, g, v[k]);
      return;
    }
    E *dst = (E *)a.vc + ((size_t)(tk[0].row / kPageTokens) * a.G + g) * kPageTokens * a.vp;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int c = head_column<NE>(i);
      if (c < a.vp)
        store4(dst + val_off(tk[0].row % kPageTokens, c, a.vp), v[0][i], v[NT > 1 ? 1 : 0][i],
               v[NT > 2 ? 2 : 0][i], v[NT > 3 ? 3 : 0][i]);
    }
    return;
  }
#pragma unroll
  for (int k = 0; k < NT; ++k) {
    if (t0 + k >= T) break;
    norm_head<NE>(a, isq, tk[k].pos, v[k]);
    if (isq) {
      E *dst = (E *)a.q + ((size_t)(t0 + k) * a.H + hd) * a.dp;
      store_head<E, NE>([&](int c) { return dst + c; }, a.dp, v[k]);
    } else {
      store_key<E, NE>(a, tk[k].row, g, v[k]);
    }
  }
}

// kRotary: a workgroup of eight waves takes NT consecutive batch tokens and every
// gridDim.y-th run of eight heads; the rows' norms first.
template <class E, int NE, int NT>
__global__ __launch_bounds__(512) void rotary_prep_kernel(const PagedToken *__restrict__ tok, int T,
                                                          AttnPrep a) {
  __shared__ float red[8][NT][2], rms[NT][2];
  const int heads = a.H + 2 * a.G, wave = threadIdx.x >> 6, lane = threadIdx.x & 63, t0 = blockIdx.x * NT;
  if (a.norms) {
    float sq[NT], sk[NT];
#pragma unroll
    for (int k = 0; k < NT; ++k) row_squares<512>(a, T, min(t0 + k, T - 1), sq[k], sk[k]);
#pragma unroll
    for (int k = 0; k < NT; ++k)
      if (lane == 0) red[wave][k][0] = sq[k], red[wave][k][1] = sk[k];
    __syncthreads();
    if (threadIdx.x < NT * 2) {
      const int k = threadIdx.x >> 1, j = threadIdx.x & 1;
      float v = 0.f;
#pragma unroll
      for (int w = 0; w < 8; ++w) v += red[w][k][j];
      rms[k][j] = inv_rms(v, (j ? a.G : a.H) * a.dim, a.eps);
    }
    __syncthreads();
  }
  PagedToken tk[NT];
#pragma unroll
  for (int k = 0; k < NT; ++k) tk[k] = tok[min(t0 + k, T - 1)];
  // four tokens in one aligned run of a page: their values lie side by side
  bool run = NT == 4 && t0 + NT <= T && tk[0].row % 4 == 0;
#pragma unroll
  for (int k = 1; k < NT; ++k) run = run && tk[k].row == tk[0].row + k;
  for (int hd = blockIdx.y * 8 + wave; hd < heads; hd += gridDim.y * 8) {
    const bool isv = hd >= a.H + a.G, isq = hd < a.H;
    const int g = isq ? 0 : (hd - a.H) % a.G;
    float v[NT][NE], bias[NE];
    load_bias<NE>(a, hd, bias);
#pragma unroll
    for (int k = 0; k < NT; ++k) load_head<NE>(a, T, min(t0 + k, T - 1), hd, bias, v[k]);
    if (isv) {
      if (a.vfreq)
#pragma unroll
        for (int k = 0; k < NT; ++k) rotate_head<NE>(a.vfreq, a.vg, 1.0f, tk[k].pos, v[k]);
      if (run) {
        E *dst = (E *)a.vc + ((size_t)(tk[0].row / kPageTokens) * a.G + g) * kPageTokens * a.vp;
#pragma unroll
        for (int i = 0; i < NE; ++i) {
          const int c = head_column<NE>(i);
          if (c < a.vp)
            store4(dst + val_off(tk[0].row % kPageTokens, c, a.vp), v[0][i], v[NT > 1 ? 1 : 0][i],
                   v[NT > 2 ? 2 : 0][i], v[NT > 3 ? 3 : 0][i]);
        }
      } else {
#pragma unroll
        for (int k = 0; k < NT; ++k)
          if (t0 + k < T) store_value<E, NE>(a, tk[k].row, g, v[k]);
      }
      continue;
    }
#pragma unroll
    for (int k = 0; k < NT; ++k) {
      if (t0 + k >= T) break;
      rotary_head<NE>(a, hd, tk[k].pos, a.norms ? rms[k][isq ? 0 : 1] : 1.0f, v[k]);
      if (isq) {
        E *dst = (E *)a.q + ((size_t)(t0 + k) * a.H + hd) * a.dp;
        store_head<E, NE>([&](int c) { return dst + c; }, a.dp, v[k]);
      } else {
        store_key<E, NE>(a, tk[k].row, g, v[k]);
      }
    }
  }
}

// ---------------------------------------------------------------------------
// attention, MFMA form
// ---------------------------------------------------------------------------
// Scores S^T = K . Q^T (a lane: 4 keys of one row), outputs O^T = V^T . P^T; the
// values' key order in the cache makes a lane's score registers the second
// product's operand as they stand, so weights never leave their lane.  Softmax
// state in fp32, base-2 exponents; weights meet the second product in bf16, the
// sums take them unrounded.
//
// Up to 16 rows (decoding, short portions): operands straight from memory, the
// workgroup's waves (eight in a step of such blocks alone, widths allowing) over half-pages, their
// results merged through LDS.
// More rows (prompts): four waves of 16 rows each over pages staged in LDS,
// double-buffered, the next page's loads in flight through registers.
//
// A lane's four keys ask for four consecutive distances: one 16-byte read of the
// bias table, issued a page ahead like the page itself.
__device__ __forceinline__ f4 bias4(const float *bh, int D, int qpos, int k0) {
  const float *p = bh + (D - min(max(qpos - k0 - 3, -4), D));
  return f4{p[0], p[1], p[2], p[3]};
}
// s = s * scale + b, keys after the query out (whole: none of the wave's are);
// the maximum taken along
template <int NK>
__device__ __forceinline__ void bias_and_mask(const f4 (&b)[NK], bool whole, int qpos, int key0,
                                              float scale, f4 (&s)[NK], float &mx) {
#pragma unroll
  for (int i = 0; i < NK; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) s[i][e] = fmaf(s[i][e], scale, b[i][e]);
  if (!whole)
#pragma unroll
    for (int i = 0; i < NK; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) s[i][e] = key0 + i * 16 + e > qpos ? -INFINITY : s[i][e];
#pragma unroll
  for (int i = 0; i < NK; ++i) mx = fmaxf(fmaxf(fmaxf(mx, s[i][0]), fmaxf(s[i][1], s[i][2])), s[i][3]);
}
// soft cap in base-2 exponents: cap tanh(s scale / cap) log2(e) with cap_in =
// 2 scale log2(e) / cap, cap_out = cap log2(e)
template <int NK>
__device__ __forceinline__ void cap_and_mask(const AttnArgs &a, bool whole, int qpos, int key0, f4 (&s)[NK],
                                             float &mx) {
  if (a.cap_in != 0.f) {
#pragma unroll
    for (int i = 0; i < NK; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float z = __builtin_amdgcn_exp2f(s[i][e] * a.cap_in) + 1.0f;
        s[i][e] = fmaf(-2.0f * a.cap_out, __builtin_amdgcn_rcpf(z), a.cap_out);
      }
  } else {
#pragma unroll
    for (int i = 0; i < NK; ++i) s[i] *= a.scale;
  }
  if (!whole)
#pragma unroll
    for (int i = 0; i < NK; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int key = key0 + i * 16 + e;
        s[i][e] = key > qpos || key <= qpos - a.window ? -INFINITY : s[i][e];
      }
#pragma unroll
  for (int i = 0; i < NK; ++i) mx = fmaxf(fmaxf(fmaxf(mx, s[i][0]), fmaxf(s[i][1], s[i][2])), s[i][3]);
}
// the factor of a row's weighted sum (maximum M, sum of weights L), the sink
// counted in
template <AttnKind KIND>
__device__ __forceinline__ float row_factor(const AttnArgs &a, int head, float M, float L) {
  if constexpr (KIND == kRotary) {
    if (a.sink) {
      const float sk = a.sink[head], top = fmaxf(M, sk), f = __builtin_amdgcn_exp2f(M - top);
      return __fdiv_rn(a.mult * f, fmaf(L, f, __builtin_amdgcn_exp2f(sk - top)));
    }
    return __fdiv_rn(a.mult, L);
  }
  return __fdiv_rn(1.0f, L);
}
// four output columns from c on: values that turned with their positions turn
// back by the query's
template <AttnKind KIND>
__device__ __forceinline__ void turn_back(const AttnArgs &a, int pos, int c, f4 &v) {
  if constexpr (KIND == kRotary) {
    if (!a.vfreq) return;
#pragma unroll
    for (int p = 0; p < 4; p += 2) {
      float cs, sn;
      turn_by(pos * a.vfreq[(c + p) >> 1], cs, sn);
      const float x = v[p], y = v[p + 1];
      v[p] = x * cs + y * sn, v[p + 1] = y * cs - x * sn;
    }
  }
}
__device__ __forceinline__ bf8 pack_weights(const f4 &lo, const f4 &hi) {
  bf8 p;
#pragma unroll
  for (int e = 0; e < 4; ++e) p[e] = (__bf16)lo[e], p[4 + e] = (__bf16)hi[e];
  return p;
}

template <int DP, int VP, int NW>
constexpr int few_rows_lds() {
  constexpr int q = 16 * (DP + 8) * 2, merge = NW * 16 * (VP + 4) * 4 + NW * 16 * 2 * 4;
  return q > merge ? q : merge;
}
template <int DP, int VP>
constexpr int attn_lds_bytes() {
  constexpr int prompt = 2 * 64 * (DP + VP) * 2;
  return prompt > few_rows_lds<DP, VP, 4>() ? prompt : few_rows_lds<DP, VP, 4>();
}

// PREP: a step of one block per request (and its splits): the workgroup first
// makes its own queries (in LDS) and, of the request's new tokens, the keys and
// values that fall into its pages; no separate launch.
template <AttnKind KIND, int DP, int VP, int NW, bool PREP>
__device__ __forceinline__ void attn_few_rows(const char *__restrict__ blob, const PagedBlock &bk,
                                              const AttnArgs &a, const AttnPrep &pr, int T,
                                              float *__restrict__ slabs, float *__restrict__ ml,
                                              char *lds) {
  constexpr int KS = DP / 32, VT = VP / 16, LDO = VP + 4;
  float *sO = reinterpret_cast<float *>(lds), *sM = sO + NW * 16 * LDO, *sL = sM + NW * 16;
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, l15 = lane & 15;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int grp = blockIdx.y, R = a.H / a.G;
  const int32_t *table = reinterpret_cast<const int32_t *>(blob) + bk.table;
  const int row = bk.row0 + min(l15, bk.nrows - 1), token = row / R, head = grp * R + row % R;
  const int qpos = bk.pos0 + token - bk.seg_row / R;
  const int qmin = bk.pos0 + (bk.row0 - bk.seg_row) / R;  // the block's first row
  const int qmax = bk.pos0 + (bk.row0 + bk.nrows - 1 - bk.seg_row) / R;
  const float *bh = KIND == kBias ? a.bias + (size_t)head * (a.D + 8) : nullptr;
  const uint16_t *Kc = (const uint16_t *)a.kc, *Vc = (const uint16_t *)a.vc;
  const int units = 2 * bk.ntiles;

  bf8 q[KS], k[2][KS], v[VT];
  f4 b[2];
  auto fetch = [&](int u) {
    const int k0 = bk.tile0 * 64 + u * 32 + 4 * g;
    if constexpr (KIND == kBias) b[0] = bias4(bh, a.D, qpos, k0), b[1] = bias4(bh, a.D, qpos, k0 + 16);
    const size_t page = (size_t)(u < 2 ? bk.page0 : table[bk.tile0 + (u >> 1)]) * a.G + grp;
    const uint16_t *kp = Kc + page * (64 * DP) + (size_t)(u & 1) * (2 * KS * 512) + lane * 8;
    const uint16_t *vp = Vc + page * (64 * VP) + (size_t)(u & 1) * (VP * 32) + l15 * 32 + g * 8;
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int ks = 0; ks < KS; ++ks)
        k[i][ks] = *reinterpret_cast<const bf8 *>(kp + (i * KS + ks) * 512);
#pragma unroll
    for (int d = 0; d < VT; ++d) v[d] = *reinterpret_cast<const bf8 *>(vp + d * 512);
  };
  if constexpr (PREP) {
    // items: the block's query rows, then a key and a value per new token
    constexpr int NE = (DP > VP ? DP : VP) / 64, LDQ = DP + 8;
    uint16_t *sQ = reinterpret_cast<uint16_t *>(lds);
    const int t0 = bk.seg_row / R, n = bk.nrows / R, nq = bk.nrows, items = nq + 2 * n;
    auto head_of = [&](int it) {
      return it < nq ? grp * R + it % R : it < nq + n ? a.H + grp : a.H + a.G + grp;
    };
    auto token_of = [&](int it) { return it < nq ? it / R : (it - nq) % n; };
    __shared__ float red[KIND == kRotary ? NW : 1][16][2], rms[16][2];
    if constexpr (KIND == kRotary)
      if (pr.norms) {  // (every group's workgroup takes the rows' norms itself)
        for (int k = 0; k < n; ++k) {
          float sq, sk;
          row_squares<NW * 64>(pr, T, t0 + k, sq, sk);
          if (lane == 0) red[wave][k][0] = sq, red[wave][k][1] = sk;
        }
        __syncthreads();
        if (tid < 2 * n) {
          const int k = tid >> 1, j = tid & 1;
          float v = 0.f;
#pragma unroll
          for (int w = 0; w < NW; ++w) v += red[w][k][j];
          rms[k][j] = inv_rms(v, (j ? pr.G : pr.H) * pr.dim, pr.eps);
        }
        __syncthreads();
      }
    auto make = [&](int it, int pos, float (&x)[NE]) {  // query or key
      if constexpr (KIND == kBias) norm_head<NE>(pr, it < nq, pos, x);
      else rotary_head<NE>(pr, head_of(it), pos, pr.norms ? rms[token_of(it)][it < nq ? 0 : 1] : 1.0f, x);
    };
    const PagedToken *ptok =
        KIND == kRotary ? reinterpret_cast<const PagedToken *>(blob + pr.off_tokens) + t0 : nullptr;
    auto conv = [&](int it, HeadConv<NE> &cv) {
      if constexpr (KIND == kRotary)
        if (pr.taps > 0) cv.load(pr, T, t0 + token_of(it), ptok[token_of(it)], head_of(it));
    };
    auto finish = [&](int it, HeadConv<NE> &cv, float (&x)[NE]) {
      const int tk = token_of(it), pos = bk.pos0 + tk, tile = pos / kPageTokens;
      if constexpr (KIND == kRotary)  // (split blocks carry the same rows)
        if (pr.taps > 0)
          cv.apply(pr, T, t0 + tk, ptok[tk], head_of(it), x);
      if (it < nq) {
        make(it, pos, x);
        store_head<uint16_t, NE>([&](int c) { return sQ + it * LDQ + c; }, DP, x);
        return;
      }
      if (tile < bk.tile0 || tile >= bk.tile0 + bk.ntiles) return;  // another workgroup's page
      const int crow = table[tile] * kPageTokens + pos % kPageTokens;
      if (it < nq + n) {
        make(it, pos, x);
        store_key<uint16_t, NE>(pr, crow, grp, x);
      } else {
        if constexpr (KIND == kBias) mix_head<NE>(pr, t0 + tk, grp, pr.vmix ? *pr.vmix : 0.f, x);
        else if (pr.vfreq) rotate_head<NE>(pr.vfreq, pr.vg, 1.0f, pos, x);
        store_value<uint16_t, NE>(pr, crow, grp, x);
      }
    };
    for (int it = wave; it < items; it += 2 * NW) {  // two at a time
      float x0[NE], x1[NE], b0[NE], b1[NE];
      const int it1 = min(it + NW, items - 1);
      load_bias<NE>(pr, head_of(it), b0);
      load_bias<NE>(pr, head_of(it1), b1);
      load_head<NE>(pr, T, t0 + token_of(it), head_of(it), b0, x0);
      load_head<NE>(pr, T, t0 + token_of(it1), head_of(it1), b1, x1);
      HeadConv<NE> c0, c1;
      conv(it, c0);
      conv(it1, c1);
      finish(it, c0, x0);
      if (it + NW < items) finish(it1, c1, x1);
    }
    __syncthreads();  // (the new keys and values are in the cache, for this workgroup)
    const uint16_t *qr = sQ + min(l15, bk.nrows - 1) * LDQ + 8 * g;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) q[ks] = *reinterpret_cast<const bf8 *>(qr + ks * 32);
    if (wave < units) fetch(wave);
    __syncthreads();  // (the merge below reuses the LDS)
  } else {
    // (the queries first: loads return in order, so the loop never waits for
    // them behind a prefetch)
    const uint16_t *qr = (const uint16_t *)a.q + ((size_t)token * a.H + head) * DP + 8 * g;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) q[ks] = *reinterpret_cast<const bf8 *>(qr + ks * 32);
    if (wave < units) fetch(wave);
  }
  f4 acc[VT];
#pragma unroll
  for (int d = 0; d < VT; ++d) acc[d] = f4{0.f, 0.f, 0.f, 0.f};
  float m = -1e30f, l = 0.f;
  for (int u = wave; u < units; u += NW) {
    f4 s[2];
    s[0] = s[1] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int i = 0; i < 2; ++i)
        s[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k[i][ks], q[ks], s[i], 0, 0, 0);
    bf8 vv[VT];
#pragma unroll
    for (int d = 0; d < VT; ++d) vv[d] = v[d];
    const f4 bb[2] = {b[0], b[1]};
    if (u + NW < units) fetch(u + NW);
    const int base = bk.tile0 * 64 + u * 32;
    float mx = -1e30f;
    if constexpr (KIND == kBias)
      bias_and_mask<2>(bb, base + 31 <= qmin, qpos, base + 4 * g, a.scale, s, mx);
    else
      cap_and_mask<2>(a, base + 31 <= qmin && base > qmax - a.window, qpos, base + 4 * g, s, mx);
    mx = fmaxf(mx, __shfl_xor(mx, 16));
    mx = fmaxf(mx, __shfl_xor(mx, 32));
    const float mn = fmaxf(m, mx), alpha = __builtin_amdgcn_exp2f(m - mn);
    m = mn;
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        s[i][e] = __builtin_amdgcn_exp2f(s[i][e] - mn);
        sum += s[i][e];
      }
    l = l * alpha + sum;
    const bf8 p = pack_weights(s[0], s[1]);
    const bool same = __all(alpha == 1.0f);
#pragma unroll
    for (int d = 0; d < VT; ++d) {
      if (!same) acc[d] *= alpha;
      acc[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vv[d], p, acc[d], 0, 0, 0);
    }
  }
  l += __shfl_xor(l, 16);
  l += __shfl_xor(l, 32);
  if (g == 0) sM[wave * 16 + l15] = m, sL[wave * 16 + l15] = l;
  __syncthreads();
  {
    float M = sM[l15];
#pragma unroll
    for (int w = 1; w < NW; ++w) M = fmaxf(M, sM[w * 16 + l15]);
    const float f = __builtin_amdgcn_exp2f(m - M);
#pragma unroll
    for (int d = 0; d < VT; ++d)
      *reinterpret_cast<f4 *>(&sO[(wave * 16 + l15) * LDO + d * 16 + 4 * g]) = acc[d] * f;
  }
  __syncthreads();
  // the waves' sums: 16 threads a row, VP / 16 columns each
  constexpr int NC = VP / 16;
  const int r = tid >> 4, c0 = (tid & 15) * NC;
  if (r >= bk.nrows) return;  // (r: 16 and above in a fifth to eighth wave)
  float M = sM[r], L = 0.f;
#pragma unroll
  for (int w = 1; w < NW; ++w) M = fmaxf(M, sM[w * 16 + r]);
#pragma unroll
  for (int w = 0; w < NW; ++w) L += sL[w * 16 + r] * __builtin_amdgcn_exp2f(sM[w * 16 + r] - M);
  f4 o[NC / 4];
#pragma unroll
  for (int c = 0; c < NC / 4; ++c) {
    o[c] = *reinterpret_cast<const f4 *>(&sO[r * LDO + c0 + c * 4]);
#pragma unroll
    for (int w = 1; w < NW; ++w)
      o[c] += *reinterpret_cast<const f4 *>(&sO[(w * 16 + r) * LDO + c0 + c * 4]);
  }
  if (bk.slot >= 0) {
    const size_t pr = ((size_t)bk.slot * a.G + grp) * 16 + r;
#pragma unroll
    for (int c = 0; c < NC / 4; ++c) *reinterpret_cast<f4 *>(slabs + pr * VP + c0 + c * 4) = o[c];
    if ((tid & 15) == 0) ml[pr * 2] = M, ml[pr * 2 + 1] = L;
    return;
  }
  const int gr = bk.row0 + r, tk = gr / R, hd = grp * R + gr % R;
  const float inv = row_factor<KIND>(a, hd, M, L);
#pragma unroll
  for (int c = 0; c < NC / 4; ++c) {
    if (c0 + c * 4 >= a.vg) continue;
    f4 v4 = o[c] * inv;
    turn_back<KIND>(a, bk.pos0 + tk - bk.seg_row / R, c0 + c * 4, v4);
    *reinterpret_cast<uint2 *>((uint16_t *)a.o + act_packed_off(tk, hd * a.vg + c0 + c * 4, a.ldo)) =
        make_uint2(f2bf(v4[0]) | ((uint32_t)f2bf(v4[1]) << 16),
                   f2bf(v4[2]) | ((uint32_t)f2bf(v4[3]) << 16));
  }
}

template <AttnKind KIND, int DP, int VP>
__device__ __forceinline__ void attn_many_rows(const char *__restrict__ blob, const PagedBlock &bk,
                                               const AttnArgs &a, float *__restrict__ slabs,
                                               float *__restrict__ ml, char *lds) {
  constexpr int KS = DP / 32, VT = VP / 16;
  uint16_t *sK = reinterpret_cast<uint16_t *>(lds), *sV = sK + 2 * 64 * DP;
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, l15 = lane & 15;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int grp = blockIdx.y, R = a.H / a.G;
  const int32_t *table = reinterpret_cast<const int32_t *>(blob) + bk.table;
  const uint16_t *Kc = (const uint16_t *)a.kc, *Vc = (const uint16_t *)a.vc;
  // this wave's rows (past the block: its last row again)
  const bool idle = wave * 16 >= bk.nrows;
  const int wrow0 = min(wave * 16, bk.nrows - 1), wrow1 = min(wave * 16 + 16, bk.nrows) - 1;
  const int qmin = bk.pos0 + (bk.row0 + wrow0 - bk.seg_row) / R;
  const int qmax = bk.pos0 + (bk.row0 + wrow1 - bk.seg_row) / R;
  const int row = bk.row0 + min(wave * 16 + l15, bk.nrows - 1);
  const int token = row / R, head = grp * R + row % R;
  const int qpos = bk.pos0 + token - bk.seg_row / R;
  const float *bh = KIND == kBias ? a.bias + (size_t)head * (a.D + 8) : nullptr;
  const float far_bias = KIND == kBias ? bh[0] : 0.f;

  // (the queries first, as above)
  bf8 q[KS];
  {
    const uint16_t *qr = (const uint16_t *)a.q + ((size_t)token * a.H + head) * DP + 8 * g;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) q[ks] = *reinterpret_cast<const bf8 *>(qr + ks * 32);
  }
  // pages are stored as their operands: staging is a straight copy
  constexpr int NKC = DP / 32, NVC = VP / 32;  // 16-byte chunks per thread
  u4 pk[NKC], pv[NVC];
  f4 pb[4];
  auto fetch = [&](int it) {
    const size_t page = (size_t)(it == 0 ? bk.page0 : table[bk.tile0 + it]) * a.G + grp;
    const u4 *kp = reinterpret_cast<const u4 *>(Kc + page * (64 * DP)) + tid;
    const u4 *vp = reinterpret_cast<const u4 *>(Vc + page * (64 * VP)) + tid;
    const int base = (bk.tile0 + it) * 64;
    if constexpr (KIND == kBias) {
#pragma unroll
      for (int j = 0; j < 4; ++j) pb[j] = f4{far_bias, far_bias, far_bias, far_bias};
      if (qmin - (base + 63) < a.D)
#pragma unroll
        for (int j = 0; j < 4; ++j) pb[j] = bias4(bh, a.D, qpos, base + j * 16 + 4 * g);
    }
#pragma unroll
    for (int i = 0; i < NKC; ++i) pk[i] = kp[i * 256];
#pragma unroll
    for (int i = 0; i < NVC; ++i) pv[i] = vp[i * 256];
  };
  auto stage = [&](int buf) {
    u4 *kd = reinterpret_cast<u4 *>(sK + buf * 64 * DP) + tid;
    u4 *vd = reinterpret_cast<u4 *>(sV + buf * 64 * VP) + tid;
#pragma unroll
    for (int i = 0; i < NKC; ++i) kd[i * 256] = pk[i];
#pragma unroll
    for (int i = 0; i < NVC; ++i) vd[i * 256] = pv[i];
  };
  fetch(0);
  f4 acc[VT];
  float m = -1e30f, l = 0.f;
#pragma unroll
  for (int d = 0; d < VT; ++d) acc[d] = f4{0.f, 0.f, 0.f, 0.f};
  stage(0);
  f4 b[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) b[j] = pb[j];
  if (bk.ntiles > 1) fetch(1);
  __syncthreads();
  for (int it = 0; it < bk.ntiles; ++it) {
    const int base = (bk.tile0 + it) * 64;
    const bool work = !idle && base <= qmax && (KIND == kBias || base + 63 > qmin - a.window);
    f4 s[4];
    if (work) {
      const uint16_t *kt = sK + (it & 1) * 64 * DP + lane * 8;
#pragma unroll
      for (int j = 0; j < 4; ++j) s[j] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        bf8 kf[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) kf[j] = *reinterpret_cast<const bf8 *>(kt + (j * KS + ks) * 512);
#pragma unroll
        for (int j = 0; j < 4; ++j)
          s[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[j], q[ks], s[j], 0, 0, 0);
      }
    }
    f4 bb[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) bb[j] = b[j];
    if (it + 1 < bk.ntiles) {
      stage((it + 1) & 1);  // (its buffer was last read before the previous barrier)
#pragma unroll
      for (int j = 0; j < 4; ++j) b[j] = pb[j];
      if (it + 2 < bk.ntiles) fetch(it + 2);
    }
    if (work) {
      const uint16_t *vt = sV + (it & 1) * 64 * VP + l15 * 32 + g * 8;
      float mx = -1e30f;
      if constexpr (KIND == kBias)
        bias_and_mask<4>(bb, base + 63 <= qmin, qpos, base + 4 * g, a.scale, s, mx);
      else
        cap_and_mask<4>(a, base + 63 <= qmin && base > qmax - a.window, qpos, base + 4 * g, s, mx);
      mx = fmaxf(mx, __shfl_xor(mx, 16));
      mx = fmaxf(mx, __shfl_xor(mx, 32));
      const float mn = fmaxf(m, mx), alpha = __builtin_amdgcn_exp2f(m - mn);
      m = mn;
      float sum = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          s[j][e] = __builtin_amdgcn_exp2f(s[j][e] - mn);
          sum += s[j][e];
        }
      l = l * alpha + sum;
      if (!__all(alpha == 1.0f))
#pragma unroll
        for (int d = 0; d < VT; ++d) acc[d] *= alpha;
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        const bf8 p = pack_weights(s[2 * h], s[2 * h + 1]);
#pragma unroll
        for (int d = 0; d < VT; ++d)
          acc[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              *reinterpret_cast<const bf8 *>(vt + h * VP * 32 + d * 512), p, acc[d], 0, 0, 0);
      }
    }
    __syncthreads();
  }
  l += __shfl_xor(l, 16);
  l += __shfl_xor(l, 32);
  const int r = wave * 16 + l15;
  if (r >= bk.nrows) return;
  if (bk.slot >= 0) {
    const size_t pr = ((size_t)(bk.slot + wave) * a.G + grp) * 16 + l15;
#pragma unroll
    for (int d = 0; d < VT; ++d) *reinterpret_cast<f4 *>(slabs + pr * VP + d * 16 + 4 * g) = acc[d];
    if (g == 0) ml[pr * 2] = m, ml[pr * 2 + 1] = l;
    return;
  }
  const float inv = row_factor<KIND>(a, head, m, l);
#pragma unroll
  for (int d = 0; d < VT; ++d) {
    const int c = d * 16 + 4 * g;
    if (c >= a.vg) continue;
    f4 v4 = acc[d] * inv;
    turn_back<KIND>(a, qpos, c, v4);
    *reinterpret_cast<uint2 *>((uint16_t *)a.o + act_packed_off(token, head * a.vg + c, a.ldo)) =
        make_uint2(f2bf(v4[0]) | ((uint32_t)f2bf(v4[1]) << 16),
                   f2bf(v4[2]) | ((uint32_t)f2bf(v4[3]) << 16));
  }
}

// MANY: the step has blocks of more than 16 rows (and maybe others)
// (256 registers a wave where the widths allow it: the accumulators then stay in
// the registers the softmax works on)
template <int VP>
constexpr int kFewWaves = VP <= 128 ? 8 : 4;
template <AttnKind KIND, int DP, int VP, bool MANY>
__global__ __launch_bounds__(MANY ? 256 : kFewWaves<VP> * 64,
                             MANY ? (DP + VP <= 256 ? 2 : 1) : kFewWaves<VP> / 4) void
paged_attn_kernel(const char *__restrict__ blob, int off_blocks, AttnArgs a, float *__restrict__ slabs,
                  float *__restrict__ ml) {
  __shared__ __attribute__((aligned(16))) char
      lds[MANY ? attn_lds_bytes<DP, VP>() : few_rows_lds<DP, VP, kFewWaves<VP>>()];
  const PagedBlock bk = reinterpret_cast<const PagedBlock *>(blob + off_blocks)[blockIdx.x];
  if (bk.nrows <= 0) return;
  if constexpr (MANY) {
    if (bk.nrows > 16) attn_many_rows<KIND, DP, VP>(blob, bk, a, slabs, ml, lds);
    else attn_few_rows<KIND, DP, VP, 4, false>(blob, bk, a, AttnPrep(), 0, slabs, ml, lds);
  } else {
    attn_few_rows<KIND, DP, VP, kFewWaves<VP>, false>(blob, bk, a, AttnPrep(), 0, slabs, ml, lds);
  }
}

// the few-rows form with its queries, keys and values made on the way
template <AttnKind KIND, int DP, int VP>
__global__ __launch_bounds__(kFewWaves<VP> * 64, kFewWaves<VP> / 4) void paged_attn_prep_kernel(
    const char *__restrict__ blob, int off_blocks, AttnArgs a, AttnPrep pr, int T,
    float *__restrict__ slabs, float *__restrict__ ml) {
  __shared__ __attribute__((aligned(16))) char lds[few_rows_lds<DP, VP, kFewWaves<VP>>()];
  const PagedBlock bk = reinterpret_cast<const PagedBlock *>(blob + off_blocks)[blockIdx.x];
  if (bk.nrows <= 0) return;
  attn_few_rows<KIND, DP, VP, kFewWaves<VP>, true>(blob, bk, a, pr, T, slabs, ml, lds);
}

// partials of split blocks, in slot order: a workgroup per 16 rows of a block
template <AttnKind KIND, int VP>
__global__ __launch_bounds__(256) void paged_attn_merge_kernel(const char *__restrict__ blob,
                                                               int off_merges, AttnArgs a,
                                                               const float *__restrict__ slabs,
                                                               const float *__restrict__ ml) {
  constexpr int NC = VP / 16, U = 4;
  const PagedMerge mg = reinterpret_cast<const PagedMerge *>(blob + off_merges)[blockIdx.x];
  const int r = blockIdx.y * 16 + (threadIdx.x >> 4), c0 = (threadIdx.x & 15) * NC;
  if (r >= mg.nrows) return;
  const int grp = blockIdx.z, R = a.H / a.G, units = mg.nrows > 16 ? kAttnTiles : 1;
  const size_t pr0 = ((size_t)(mg.slot0 + blockIdx.y) * a.G + grp) * 16 + (r & 15);
  const size_t step = (size_t)units * a.G * 16;
  float M = -1e30f;
  for (int i = 0; i < mg.nslots; ++i) M = fmaxf(M, ml[(pr0 + i * step) * 2]);
  float L = 0.f;
  f4 o[NC / 4];
#pragma unroll
  for (int c = 0; c < NC / 4; ++c) o[c] = f4{0.f, 0.f, 0.f, 0.f};
  for (int i0 = 0; i0 < mg.nslots; i0 += U) {
    f4 v[U][NC / 4];
    float w[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const size_t pr = pr0 + min(i0 + u, mg.nslots - 1) * step;
      w[u] = i0 + u < mg.nslots ? __builtin_amdgcn_exp2f(ml[pr * 2] - M) : 0.f;
      L = fmaf(w[u], ml[pr * 2 + 1], L);
#pragma unroll
      for (int c = 0; c < NC / 4; ++c) v[u][c] = *reinterpret_cast<const f4 *>(slabs + pr * VP + c0 + c * 4);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int c = 0; c < NC / 4; ++c) o[c] += v[u][c] * w[u];
  }
  const int gr = mg.row0 + r, tk = gr / R, hd = grp * R + gr % R;
  const float inv = row_factor<KIND>(a, hd, M, L);
  const int pos = KIND == kRotary ? reinterpret_cast<const PagedToken *>(blob + a.off_tokens)[tk].pos : 0;
#pragma unroll
  for (int c = 0; c < NC / 4; ++c) {
    if (c0 + c * 4 >= a.vg) continue;
    f4 v4 = o[c] * inv;
    turn_back<KIND>(a, pos, c0 + c * 4, v4);
    *reinterpret_cast<uint2 *>((uint16_t *)a.o + act_packed_off(tk, hd * a.vg + c0 + c * 4, a.ldo)) =
        make_uint2(f2bf(v4[0]) | ((uint32_t)f2bf(v4[1]) << 16),
                   f2bf(v4[2]) | ((uint32_t)f2bf(v4[3]) << 16));
  }
}

template <AttnKind KIND, int DP, int VP>
static hipError_t run_paged_attn(const char *blob, const PagedLists &pl, const AttnArgs &a,
                                 const AttnPrep *pr, int T, float *slabs, float *ml, hipStream_t s) {
  const dim3 grid(pl.num_blocks, a.G);
  if (pr)
    hipLaunchKernelGGL((paged_attn_prep_kernel<KIND, DP, VP>), grid, dim3(kFewWaves<VP> * 64), 0, s, blob,
                       pl.off_blocks, a, *pr, T, slabs, ml);
  else if (pl.row_tiles > 1)
    hipLaunchKernelGGL((paged_attn_kernel<KIND, DP, VP, true>), grid, dim3(256), 0, s, blob, pl.off_blocks, a,
                       slabs, ml);
  else
    hipLaunchKernelGGL((paged_attn_kernel<KIND, DP, VP, false>), grid, dim3(kFewWaves<VP> * 64), 0, s, blob,
                       pl.off_blocks, a, slabs, ml);
  if (pl.num_merges > 0)
    hipLaunchKernelGGL((paged_attn_merge_kernel<KIND, VP>), dim3(pl.num_merges, pl.row_tiles, a.G), dim3(256),
                       0, s, blob, pl.off_merges, a, slabs, ml);
  return hipGetLastError();
}

template <AttnKind KIND>
static hipError_t launch_attn_kind(const char *blob, const PagedLists &pl, AttnArgs a, float *slabs,
                                   float *ml, hipStream_t s, const AttnPrep *pr, int T) {
  if (pl.num_blocks <= 0) return hipSuccess;
  if (!a.ldo) a.ldo = a.H * a.vg;
  if (pr && pr->taps > 0 && (KIND != kRotary || !pr->conv || (pr->taps > 1 && !pr->carry)))
    return hipErrorInvalidValue;
  if (pr && (pl.row_tiles != 1 || pr->H != a.H || pr->G != a.G || pr->dp != a.dp || pr->vp != a.vp ||
             pr->vg != a.vg || pr->y.S < 1 || pr->y.S > 8 || pr->every < 1))
    return hipErrorInvalidValue;
  if (a.G < 1 || a.H % a.G || pl.heads != a.H / a.G || pl.groups != a.G || a.vg > a.vp || a.D < 0 ||
      a.ldo < a.H * a.vg || a.ldo % 32 || a.window < 1 || (pl.window && pl.window != a.window) ||
      (pl.row_tiles != 1 && pl.row_tiles != kAttnTiles))
    return hipErrorInvalidValue;
#define FFMI_PA(DP, VP) \
  if (a.dp == DP && a.vp == VP) return run_paged_attn<KIND, DP, VP>(blob, pl, a, pr, T, slabs, ml, s)
  FFMI_PA(64, 64);
  FFMI_PA(64, 128);
  FFMI_PA(64, 256);
  FFMI_PA(128, 64);
  FFMI_PA(128, 128);
  FFMI_PA(128, 256);
  FFMI_PA(256, 64);
  FFMI_PA(256, 128);
  FFMI_PA(256, 256);
#undef FFMI_PA
  return hipErrorInvalidValue;
}

// ---------------------------------------------------------------------------
// attention, one workgroup per row (fp32, and bf16 widths without an MFMA form)
// ---------------------------------------------------------------------------
template <AttnKind KIND, class E>
__global__ __launch_bounds__(256) void paged_attn_rows_kernel(const char *__restrict__ blob,
                                                              int off_blocks, AttnArgs a) {
  __shared__ float sq[kAttnRowsMax], sp[256], red[4];
  __shared__ int spage[256];
  const PagedBlock bk = reinterpret_cast<const PagedBlock *>(blob + off_blocks)[blockIdx.x];
  const int r = blockIdx.y, tid = threadIdx.x, grp = blockIdx.z, R = a.H / a.G;
  if (r >= bk.nrows) return;
  const int32_t *table = reinterpret_cast<const int32_t *>(blob) + bk.table;
  const int row = bk.row0 + r, token = row / R, head = grp * R + row % R;
  const int qpos = bk.pos0 + token - bk.seg_row / R, n = qpos + 1;
  const int first = KIND == kRotary ? max(0, n - a.window) : 0;
  const float *bh = KIND == kBias ? a.bias + (size_t)head * (a.D + 8) : nullptr;
  const E *q = (const E *)a.q + ((size_t)token * a.H + head) * a.dp;
  for (int i = tid; i < a.dp; i += 256) sq[i] = ld_elem(q + i);
  float acc[kAttnRowsMax / 256];
#pragma unroll
  for (int i = 0; i < kAttnRowsMax / 256; ++i) acc[i] = 0.f;
  constexpr bool base2 = sizeof(E) == 2;
  float m = -1e30f, l = 0.f;
  for (int j0 = first; j0 < n; j0 += 256) {
    __syncthreads();
    const int j = j0 + tid;
    float sv = -INFINITY;
    if (j < n) {
      const int page = table[j >> 6] * a.G + grp;
      spage[tid] = page;
      const E *k = (const E *)a.kc + (size_t)page * (64 * a.dp);
      float d = 0.f;
      for (int c = 0; c < a.dp; c += 8) {
        const E *kc = k + key_off(j & 63, c, a.dp);
#pragma unroll
        for (int e = 0; e < 8; ++e) d = fmaf(sq[c + e], ld_elem(kc + e), d);
      }
      if constexpr (KIND == kBias) sv = fmaf(d, a.scale, bh[a.D + 3 - min(qpos - j, a.D)]);
      else if (a.cap_in == 0.f) sv = d * a.scale;
      else sv = a.cap_out * tanhf(d * a.cap_in * (base2 ? 0.34657359028f : 1.0f));
    }
    float mx = sv;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o));
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    const float mn = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float p = j < n ? (base2 ? exp2f(sv - mn) : expf(sv - mn)) : 0.f;
    sp[tid] = p;
    float sum = p;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) sum += __shfl_xor(sum, o);
    __syncthreads();
    if ((tid & 63) == 0) red[tid >> 6] = sum;
    __syncthreads();
    const float al = base2 ? exp2f(m - mn) : expf(m - mn);
    l = l * al + (red[0] + red[1] + red[2] + red[3]);
    m = mn;
    const int cnt = min(256, n - j0);
#pragma unroll
    for (int i = 0; i < kAttnRowsMax / 256; ++i) {
      const int c = tid + i * 256;
      if (c >= a.vg) break;
      float s = acc[i] * al;
      for (int k = 0; k < cnt; ++k)
        s = fmaf(sp[k], ld_elem((const E *)a.vc + (size_t)spage[k] * (64 * a.vp) +
                                val_off((j0 + k) & 63, c, a.vp)), s);
      acc[i] = s;
    }
  }
  float inv = __fdiv_rn(KIND == kRotary ? a.mult : 1.0f, l);
  if constexpr (KIND == kRotary)
    if (a.sink) {
      const float sk = a.sink[head], top = fmaxf(m, sk);
      const float f = base2 ? exp2f(m - top) : expf(m - top);
      inv = __fdiv_rn(a.mult * f, l * f + (base2 ? exp2f(sk - top) : expf(sk - top)));
    }
#pragma unroll
  for (int i = 0; i < kAttnRowsMax / 256; ++i) {
    const int c = tid + i * 256, col = head * a.vg + c;
    float v = acc[i] * inv;
    if constexpr (KIND == kRotary)
      if (a.vfreq) {
        const float other = __shfl_xor(v, 1);
        float cs, sn;
        turn_by(qpos * a.vfreq[min(c, a.vg - 1) >> 1], cs, sn);
        v = c & 1 ? v * cs - other * sn : v * cs + other * sn;
      }
    if (c >= a.vg) break;
    st_elem((E *)a.o + (base2 ? act_packed_off(token, col, a.ldo) : (size_t)token * a.ldo + col), v);
  }
}

template <AttnKind KIND>
static hipError_t launch_attn_rows_kind(const char *blob, const PagedLists &pl, AttnArgs a, bool f32,
                                        hipStream_t s) {
  if (pl.num_blocks <= 0) return hipSuccess;
  if (!a.ldo) a.ldo = a.H * a.vg;
  if (a.G < 1 || a.H % a.G || pl.heads != a.H / a.G || pl.groups != a.G || a.dp > kAttnRowsMax ||
      a.vp > kAttnRowsMax || a.dp % 32 || a.vg > a.vp || a.D < 0 || pl.num_merges > 0 || a.window < 1 ||
      a.ldo < a.H * a.vg || a.ldo % 32)
    return hipErrorInvalidValue;
  const dim3 grid(pl.num_blocks, pl.row_tiles * 16, a.G);
  if (f32)
    hipLaunchKernelGGL((paged_attn_rows_kernel<KIND, float>), grid, dim3(256), 0, s, blob, pl.off_blocks, a);
  else
    hipLaunchKernelGGL((paged_attn_rows_kernel<KIND, uint16_t>), grid, dim3(256), 0, s, blob, pl.off_blocks, a);
  return hipGetLastError();
}

}  // namespace ffmi
