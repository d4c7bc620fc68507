// conv_norm.hip -- sums of parallel sublayers, group norm, causal convolution
// (conv_norm.h).
#include "conv_norm.h"

#include <algorithm>

#include "device_util.h"

namespace ffmi {

struct ConvNormStep {
  const char *blob = nullptr;
  uint4 *blob_dst = nullptr;  // null: nothing to copy
  int blob_n16 = 0, off_tokens = 0, T = 0;
  const int32_t *out_rows = nullptr;  // null: all tokens
  int unit = 8, parts = 0;  // columns of a partial sum, partials of a row
  bool waves = false;       // (unit 512: a partial per wave and chunk)
};

// A workgroup takes a token; a thread has chunks of 8 columns.  Few tokens (CONV):
// the convolution as well; the rows h that it reads are made again from x_in (so x
// and x_in are different buffers), after the token's own, or come from `carry`.  Many
// tokens: conv_kernel follows, on the x and inv of this one.
// MAXS == 0: x is an embedding row.
// REGS: the earlier rows are kept in registers (taps <= 4), else in LDS, each thread
// its own.
template <int NT, int MAXC, int MAXS, bool CONV, bool REGS>
__global__ __launch_bounds__(NT) void conv_norm_kernel(ConvNormStep st, ConvNorm a, EmbedPairs em) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, H = a.H, nchunk = H >> 3, T = st.T;
  const PagedToken *tok = reinterpret_cast<const PagedToken *>(st.blob + st.off_tokens);
  const int first = st.out_rows ? st.out_rows[blockIdx.x] : (int)blockIdx.x;
  const int out = blockIdx.x;
  const PagedToken raw = tok[first];  // (one token for the whole workgroup)
  if (st.blob_dst) {
    const uint4 *src = reinterpret_cast<const uint4 *>(st.blob);
    for (int i = blockIdx.x * NT + tid; i < st.blob_n16; i += gridDim.x * NT) st.blob_dst[i] = src[i];
  }
  const int gs = a.n / a.groups, per = st.waves ? (gs + 511) / 512 : gs / st.unit;
  float *part = lds, *inv = lds + 2 * st.parts;
  f4 *ring = reinterpret_cast<f4 *>(lds + ((2 * st.parts + a.groups + 3) & ~3));
  const int past = CONV ? a.taps - 1 : 0;
  auto chunk = [&](int c) { return min(tid + c * NT, nchunk - 1); };
  auto load8 = [](const float *p, f4 (&v)[2]) {
    v[0] = *reinterpret_cast<const f4 *>(p), v[1] = *reinterpret_cast<const f4 *>(p + 4);
  };
  // the row k + 1 tokens back
  constexpr int KH = REGS ? 3 : 1;
  f4 hist[KH][MAXC][2];
  int head = 0;  // (LDS) slot of the latest row
  auto ring_at = [&](int slot, int c, int h) -> f4 & { return ring[(slot * 2 + h) * nchunk + chunk(c)]; };
  auto old_row = [&](int k, int c, int h) {
    if constexpr (REGS) return hist[k][c][h];
    return ring_at(head - k < 0 ? head - k + past : head - k, c, h);
  };
  // x of row t; meanwhile() runs while its first loads are under way
  auto sum_row = [&](int t, auto meanwhile, f4 (&x)[MAXC][2]) {
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      const int ch = chunk(c);
      if constexpr (MAXS == 0) {
        PagedToken tk = t == first ? raw : tok[t];
        const int token = __builtin_amdgcn_readfirstlane(tk.token), prev = __builtin_amdgcn_readfirstlane(tk.prev);
        unpack8_bf16(*reinterpret_cast<const uint4 *>(em.embed + (size_t)token * H + ch * 8), x[c][0], x[c][1]);
        f4 p[2];
        p[0] = p[1] = f4{0.f, 0.f, 0.f, 0.f};
        if (em.pairs) {
          const int64_t b = prev < 0 ? em.buckets : (prev * em.mul_prev + token * em.mul_cur) % em.buckets;
          unpack8_bf16(*reinterpret_cast<const uint4 *>(em.pairs + (size_t)b * H + ch * 8), p[0], p[1]);
        }
        if (c == 0) meanwhile();
#pragma unroll
        for (int h = 0; h < 2; ++h) x[c][h] = x[c][h] * em.scale + p[h];
      } else {
        constexpr int SB = MAXC > 1 ? 1 : NT > 512 ? (MAXS < 2 ? 1 : 2) : (MAXS < 1 ? 1 : MAXS);  // slabs in flight
        constexpr int U = MAXC > 1 ? 1 : NT > 512 ? 2 : 4;                                      // expert rows
        f4 y[2], s[SB][2];
        const int32_t *at = a.at + (size_t)t * a.top;
        const float *wt = a.wt + (size_t)t * a.top;
        int at0[U];
        float wt0[U];
        if (a.rows)
#pragma unroll
          for (int k = 0; k < U; ++k) at0[k] = at[min(k, a.top - 1)], wt0[k] = wt[min(k, a.top - 1)];
        load8(a.x_in + (size_t)t * H + ch * 8, x[c]);
        y[0] = y[1] = f4{0.f, 0.f, 0.f, 0.f};
        const float *p = a.y.p + (size_t)t * a.y.NP + ch * 8;
        if (a.y.S > 0)
#pragma unroll
          for (int sl = 0; sl < SB; ++sl) load8(p + (size_t)min(sl, a.y.S - 1) * T * a.y.NP, s[sl]);
        if (c == 0) meanwhile();
        if (a.y.S > 0) {
#pragma unroll
          for (int s0 = 0; s0 < MAXS; s0 += SB) {
            if (s0 >= a.y.S) break;
            if (s0 > 0)
#pragma unroll
              for (int sl = 0; sl < SB; ++sl) load8(p + (size_t)min(s0 + sl, a.y.S - 1) * T * a.y.NP, s[sl]);
#pragma unroll
            for (int sl = 0; sl < SB; ++sl)
              if (s0 + sl < a.y.S) y[0] += s[sl][0], y[1] += s[sl][1];
          }
        }
        if (a.rows) {
          for (int k0 = 0; k0 < a.top; k0 += U) {
            f4 r[U][2];
            float w4[U];
#pragma unroll
            for (int k = 0; k < U; ++k) {
              const int kk = min(k0 + k, a.top - 1);
              const size_t o = (size_t)(k0 ? at[kk] : at0[k]) * H + ch * 8;
              w4[k] = k0 + k >= a.top ? 0.f : k0 ? wt[kk] : wt0[k];
              if (a.rows_f32) load8((const float *)a.rows + o, r[k]);
              else unpack8_bf16(*reinterpret_cast<const uint4 *>((const uint16_t *)a.rows + o), r[k][0], r[k][1]);
            }
#pragma unroll
            for (int k = 0; k < U; ++k) y[0] += r[k][0] * w4[k], y[1] += r[k][1] * w4[k];
          }
        }
#pragma unroll
        for (int h = 0; h < 2; ++h) x[c][h] += y[h] * a.mult;
      }
    }
  };
  // 1 / rms of every column's group, of row t
  auto group_rms = [&](int t, int odd, const f4 (&x)[MAXC][2], f4 (&r)[MAXC][2]) {
    float ss[MAXC];
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      ss[c] = 0.f;
      if (tid + c * NT < nchunk)
#pragma unroll
        for (int e = 0; e < 8; ++e) ss[c] = fmaf(x[c][e >> 2][e & 3], x[c][e >> 2][e & 3], ss[c]);
    }
    if (st.waves) {  // a wave's 512 columns lie in one group
      float *pb = part + odd * st.parts;
#pragma unroll
      for (int c = 0; c < MAXC; ++c) {
        float v = ss[c];
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
        const int u = wave + c * (NT / 64);
        if (lane == 0 && u < st.parts) pb[u] = v;
      }
      __syncthreads();
#pragma unroll
      for (int c = 0; c < MAXC; ++c) {
        const int u0 = wave + c * (NT / 64), g = min(u0 / per, a.groups - 1);
        float v = 0.f;
        for (int u = 0; u < per; ++u) v += pb[g * per + u];
        v = inv_rms(v, gs, a.eps);
        if (!CONV && a.inv && lane == 0 && u0 < st.parts && u0 % per == 0) a.inv[(size_t)t * a.groups + g] = v;
        r[c][0] = r[c][1] = f4{v, v, v, v};
      }
      return;
    }
    const int us = st.unit, np = 8 / us;
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      const int ch = tid + c * NT;
      if (ch >= nchunk) continue;
      if (us == 8) {
        if (ch < st.parts) part[ch] = ss[c];
        continue;
      }
      int u = ch * np;
      float v = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) {  // (us divides 8: runs of us columns)
        v = fmaf(x[c][e >> 2][e & 3], x[c][e >> 2][e & 3], v);
        if ((e + 1) & (us - 1)) continue;
        if (u < st.parts) part[u] = v;
        ++u, v = 0.f;
      }
    }
    __syncthreads();
    for (int g = wave; g < a.groups; g += NT / 64) {
      float v = 0.f;
      for (int u = lane; u < per; u += 64) v += part[g * per + u];
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
      if (lane == 0) {
        inv[g] = inv_rms(v, gs, a.eps);
        if (!CONV && a.inv) a.inv[(size_t)t * a.groups + g] = inv[g];
      }
    }
    __syncthreads();
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      const int ch = chunk(c);
      int g = ch * 8 / gs, next = (g + 1) * gs;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        if (ch * 8 + e >= next) ++g, next += gs;
        r[c][e >> 2][e & 3] = inv[min(g, a.groups - 1)];
      }
    }
  };

  int pos = 0, back = 0, ahead = 0, bank = 0;
  size_t slot = 0;
  // rows of earlier steps, zeros before the sequence (read while the token's own
  // row is summed)
  auto carried = [&]() {
    if constexpr (!CONV) return;
    pos = __builtin_amdgcn_readfirstlane(raw.pos), back = __builtin_amdgcn_readfirstlane(raw.back);
    ahead = __builtin_amdgcn_readfirstlane(raw.ahead), bank = __builtin_amdgcn_readfirstlane(raw.bank);
    slot = __builtin_amdgcn_readfirstlane(raw.slot);
    if (past == 0 || back > past) return;
    const float *cr = a.carry + (slot * 2 + bank) * past * H;
    for (int k = 0; k < (REGS ? 1 : past); ++k)
#pragma unroll
      for (int kr = 0; kr < KH; ++kr)
#pragma unroll
        for (int c = 0; c < MAXC; ++c) {
          const int q = REGS ? kr : k;
          f4 v[2];
          v[0] = v[1] = f4{0.f, 0.f, 0.f, 0.f};
          if (q < past && pos - back > q) load8(cr + (size_t)q * H + chunk(c) * 8, v);
#pragma unroll
          for (int h = 0; h < 2; ++h) {
            if constexpr (REGS) hist[kr][c][h] = v[h];
            else if (tid + c * NT < nchunk) ring_at(q ? past - q : 0, c, h) = v[h];
          }
        }
  };
  f4 hown[MAXC][2], w[MAXC][2];
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    w[c][0] = w[c][1] = f4{0.f, 0.f, 0.f, 0.f};
    if (a.w) load8(a.w + chunk(c) * 8, w[c]);
  }
  {
    f4 r[MAXC][2];
    sum_row(first, carried, hown);
#pragma unroll
    for (int c = 0; c < MAXC; ++c)
#pragma unroll
      for (int h = 0; h < 2; ++h)
        if (a.x && tid + c * NT < nchunk)
          *reinterpret_cast<f4 *>(a.x + (size_t)first * H + (tid + c * NT) * 8 + 4 * h) = hown[c][h];
    if (!a.w) return;
    group_rms(first, 0, hown, r);
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
#pragma unroll
      for (int h = 0; h < 2; ++h) hown[c][h] = hown[c][h] * r[c][h] * w[c][h];
      const int ch = tid + c * NT;
      if (ch >= nchunk) continue;
      const uint4 hp = pack8_bf16(hown[c][0], hown[c][1]);
      if (a.hb) *reinterpret_cast<uint4 *>(a.hb + act_packed_off(out, ch * 8, H)) = hp;
      if (a.hrow) *reinterpret_cast<uint4 *>(a.hrow + (size_t)out * H + ch * 8) = hp;
      if (a.hf) {
        *reinterpret_cast<f4 *>(a.hf + (size_t)out * H + ch * 8) = hown[c][0];
        *reinterpret_cast<f4 *>(a.hf + (size_t)out * H + ch * 8 + 4) = hown[c][1];
      }
    }
  }
  if constexpr (CONV) {
    // the rows before it that this step brought, oldest first
    for (int t = first - min(back, past), odd = 1; t < first; ++t, odd ^= 1) {
      f4 x[MAXC][2], r[MAXC][2];
      sum_row(t, []() {}, x);
      group_rms(t, odd, x, r);
      if constexpr (!REGS) head = head + 1 == past ? 0 : head + 1;
#pragma unroll
      for (int c = 0; c < MAXC; ++c)
#pragma unroll
        for (int h = 0; h < 2; ++h) {
          const f4 v = x[c][h] * r[c][h] * w[c][h];
          if constexpr (REGS) hist[2][c][h] = hist[1][c][h], hist[1][c][h] = hist[0][c][h], hist[0][c][h] = v;
          else if (tid + c * NT < nchunk) ring_at(head, c, h) = v;
        }
    }
    const bool last = ahead == 0;
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      const int ch = tid + c * NT;
      if (ch >= nchunk) continue;
      f4 cv[2];
      float *cr = a.carry + ((slot * 2 + (bank ^ 1)) * past) * H + ch * 8;
      const float *cw = a.conv + ch * 8;
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        // (oldest first, the token's own tap last)
        f4 v = f4{0.f, 0.f, 0.f, 0.f};
        if constexpr (REGS) {
#pragma unroll
          for (int k = 2; k >= 0; --k)
            if (k < past) {
              v += hist[k][c][h] * *reinterpret_cast<const f4 *>(cw + (size_t)(past - 1 - k) * H + 4 * h);
              if (last && k + 1 < past) *reinterpret_cast<f4 *>(cr + (size_t)(k + 1) * H + 4 * h) = hist[k][c][h];
            }
        } else {
          for (int k = past - 1; k >= 0; --k) {
            const f4 o = old_row(k, c, h);
            v += o * *reinterpret_cast<const f4 *>(cw + (size_t)(past - 1 - k) * H + 4 * h);
            if (last && k + 1 < past) *reinterpret_cast<f4 *>(cr + (size_t)(k + 1) * H + 4 * h) = o;
          }
        }
        v += hown[c][h] * *reinterpret_cast<const f4 *>(cw + (size_t)past * H + 4 * h);
        if (last && past > 0) *reinterpret_cast<f4 *>(cr + 4 * h) = hown[c][h];
        cv[h] = hown[c][h] + v;
      }
      if (a.cb) *reinterpret_cast<uint4 *>(a.cb + act_packed_off(out, ch * 8, H)) = pack8_bf16(cv[0], cv[1]);
      if (a.cf) {
        *reinterpret_cast<f4 *>(a.cf + (size_t)out * H + ch * 8) = cv[0];
        *reinterpret_cast<f4 *>(a.cf + (size_t)out * H + ch * 8 + 4) = cv[1];
      }
    }
  }
}

// The convolution of many tokens: a thread has 4 columns of C consecutive tokens,
// a workgroup 4 C tokens side by side (16: whole lines of the packed tiles).
// TAPS: at most (0: any; earlier rows are then read for every token again).
template <int C, int TAPS>
__global__ __launch_bounds__(256) void conv_kernel(const PagedToken *__restrict__ tok, int T, ConvNorm a) {
  const int H = a.H, past = a.taps - 1, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int col = (blockIdx.y * 64 + lane) * 4, t0 = (blockIdx.x * 4 + wave) * C;
  if (col >= H || t0 >= T) return;
  const int gs = a.n / a.groups, g0 = min(col / gs, a.groups - 1);
  const bool one = min((col + 3) / gs, a.groups - 1) == g0;  // (else the columns lie in several groups)
  auto load4 = [](const float *p) { return *reinterpret_cast<const f4 *>(p); };
  const f4 w = load4(a.w + col), own = load4(a.conv + (size_t)past * H + col);
  auto inv_of = [&](int t) {
    const float *iv = a.inv + (size_t)t * a.groups;
    const float r = iv[g0];
    f4 v = {r, r, r, r};
    if (!one)
#pragma unroll
      for (int e = 1; e < 4; ++e) v[e] = iv[min((col + e) / gs, a.groups - 1)];
    return v;
  };
  auto carry_at = [&](const PagedToken &tk, int bank, int q) {
    return a.carry + ((size_t)(tk.slot * 2 + bank) * past + q) * H + col;
  };
  // the row of q + 1 tokens before the step's first one of the request
  auto old_row = [&](const PagedToken &tk, int q) {
    return tk.pos - tk.back > q ? load4(carry_at(tk, tk.bank, q)) : f4{0.f, 0.f, 0.f, 0.f};
  };
  auto keep = [&](const PagedToken &tk, int q, const f4 &h) {
    if (tk.ahead == 0 && q < past) *reinterpret_cast<f4 *>(carry_at(tk, tk.bank ^ 1, q)) = h;
  };
  auto finish = [&](int t, const PagedToken &tk, const f4 &h, f4 v) {
    keep(tk, 0, h);
    v = h + (v + h * own);
    if (a.cb)
      *reinterpret_cast<uint2 *>(a.cb + act_packed_off(t, col, H)) =
          make_uint2(f2bf(v[0]) | ((uint32_t)f2bf(v[1]) << 16), f2bf(v[2]) | ((uint32_t)f2bf(v[3]) << 16));
    if (a.cf) *reinterpret_cast<f4 *>(a.cf + (size_t)t * H + col) = v;
  };
  if constexpr (TAPS > 0) {
    constexpr int P = TAPS - 1;
    f4 h[C + P], r[C + P], cw[P];  // rows t0 - P .., taps of the rows 1 to P tokens back
    PagedToken tk[C];
#pragma unroll
    for (int i = 0; i < C + P; ++i) {
      const int t = min(max(t0 - P + i, 0), T - 1);
      h[i] = load4(a.x + (size_t)t * H + col), r[i] = inv_of(t);
    }
#pragma unroll
    for (int k = 0; k < P; ++k) cw[k] = load4(a.conv + (size_t)max(past - 1 - k, 0) * H + col);
#pragma unroll
    for (int i = 0; i < C; ++i) tk[i] = tok[min(t0 + i, T - 1)];
#pragma unroll
    for (int i = 0; i < C + P; ++i) h[i] = h[i] * r[i] * w;
#pragma unroll
    for (int i = 0; i < C; ++i) {
      if (t0 + i >= T) break;
      f4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = P - 1; k >= 0; --k)  // (oldest first, the token's own tap last)
        if (k < past) {
          const f4 o = tk[i].back > k ? h[i + P - 1 - k] : old_row(tk[i], k - tk[i].back);
          v += o * cw[k];
          keep(tk[i], k + 1, o);
        }
      finish(t0 + i, tk[i], h[i + P], v);
    }
  } else {
    for (int t = t0; t < min(t0 + C, T); ++t) {
      const PagedToken tk = tok[t];
      f4 v = {0.f, 0.f, 0.f, 0.f};
      for (int k = past - 1; k >= 0; --k) {
        const int s = t - 1 - k;
        const f4 o = tk.back > k ? load4(a.x + (size_t)s * H + col) * inv_of(s) * w : old_row(tk, k - tk.back);
        v += o * load4(a.conv + (size_t)(past - 1 - k) * H + col);
        keep(tk, k + 1, o);
      }
      finish(t, tk, load4(a.x + (size_t)t * H + col) * inv_of(t) * w, v);
    }
  }
}

// steps of more tokens take the convolution from a launch of its own
constexpr int kConvFused = 64;
static hipError_t run_conv_norm(ConvNormStep st, const ConvNorm &a, const EmbedPairs &em, int blocks,
                                hipStream_t s) {
  const int nchunk = a.H / 8;
  if (a.H % 32 || a.n > a.H || a.groups < 1 || a.n % a.groups || a.y.S < 0 || a.y.S > 8) return hipErrorInvalidValue;
  if (a.y.S > 0 && (a.y.NP < a.H || a.y.NP % 4 || !a.y.p)) return hipErrorInvalidValue;
  if (a.rows && (!a.at || !a.wt || a.top < 1)) return hipErrorInvalidValue;
  if (!em.embed && (!a.x_in || a.x_in == a.x)) return hipErrorInvalidValue;
  if (a.conv && (!a.w || a.taps < 1 || (a.taps > 1 && !a.carry))) return hipErrorInvalidValue;
  // many tokens: the convolution in a launch of its own
  const bool split = a.conv && st.T > kConvFused && a.x && a.inv, conv = a.conv && !split;
  const int gs = a.n / a.groups;
  st.waves = a.groups == 1 || gs % 512 == 0;
  st.unit = st.waves ? 512 : gs % 8 == 0 ? 8 : gs % 4 == 0 ? 4 : gs % 2 == 0 ? 2 : 1;
  st.parts = st.waves ? (a.n + 511) / 512 : a.n / st.unit;
  const bool regs = conv && a.taps <= 4 && nchunk <= 1024;  // (wider rows: in LDS)
  size_t lds = (size_t)((2 * st.parts + a.groups + 3) & ~3) * 4;
  if (conv && !regs) lds += (size_t)(a.taps - 1) * a.H * 4;
  if (lds > 160 * 1024) return hipErrorInvalidValue;
#define FFMI_CN2(NT, MC, MS, CV, RG)                                                                   \
  do {                                                                                                 \
    if (lds > 64 * 1024) {                                                                             \
      const hipError_t e = hipFuncSetAttribute((const void *)(conv_norm_kernel<NT, MC, MS, CV, RG>),   \
                                               hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); \
      if (e != hipSuccess) return e;                                                                   \
    }                                                                                                  \
    hipLaunchKernelGGL((conv_norm_kernel<NT, MC, MS, CV, RG>), dim3(blocks), dim3(NT), lds, s, st, a, em); \
  } while (0)
#define FFMI_CN1(NT, MC, MS)                                   \
  do {                                                         \
    if (!conv) FFMI_CN2(NT, MC, MS, false, false);             \
    else if (MC == 1 && regs) FFMI_CN2(NT, MC, MS, true, (MC == 1)); \
    else FFMI_CN2(NT, MC, MS, true, false);                    \
  } while (0)
#define FFMI_CN(NT, MC)                                         \
  do {                                                          \
    if (em.embed) FFMI_CN1(NT, MC, 0);                          \
    else if (MC == 1 && a.y.S <= 2) FFMI_CN1(NT, MC, (MC == 1 ? 2 : 8)); \
    else FFMI_CN1(NT, MC, 8);                                   \
  } while (0)
  if (nchunk <= 128) FFMI_CN(128, 1);
  else if (nchunk <= 256) FFMI_CN(256, 1);
  else if (nchunk <= 512) FFMI_CN(512, 1);
  else if (nchunk <= 1024) FFMI_CN(1024, 1);
  else if (nchunk <= 2048) FFMI_CN(1024, 2);
  else return hipErrorInvalidValue;
#undef FFMI_CN
#undef FFMI_CN1
#undef FFMI_CN2
  if (split) {
    // (the first kernel's staging copy is there by now, in any form)
    const PagedToken *tok =
        reinterpret_cast<const PagedToken *>((st.blob_dst ? (const char *)st.blob_dst : st.blob) + st.off_tokens);
#define FFMI_CV(C, TP) \
  hipLaunchKernelGGL((conv_kernel<C, TP>), dim3((st.T + 4 * C - 1) / (4 * C), (a.H / 4 + 63) / 64), dim3(256), 0, s, tok, st.T, a)
    if (a.taps <= 4) FFMI_CV(4, 4);
    else FFMI_CV(4, 0);
#undef FFMI_CV
  }
  return hipGetLastError();
}

hipError_t launch_conv_norm(const char *blob_src, char *blob_dst, size_t blob_bytes, int off_tokens,
                            const ConvNorm &a, const EmbedPairs *em, int T, hipStream_t s) {
  if (T <= 0) return hipSuccess;
  if (em && off_tokens) return hipErrorInvalidValue;
  ConvNormStep st;
  st.blob = blob_src, st.off_tokens = off_tokens, st.T = T;
  if (em) st.blob_dst = reinterpret_cast<uint4 *>(blob_dst), st.blob_n16 = (int)((blob_bytes + 15) / 16);
  return run_conv_norm(st, a, em ? *em : EmbedPairs(), T, s);
}

hipError_t launch_conv_norm_rows(const char *blob, int off_tokens, int off_rows, const ConvNorm &a, int T,
                                 int R, hipStream_t s) {
  if (R <= 0) return hipSuccess;
  if (a.conv || a.x) return hipErrorInvalidValue;
  ConvNormStep st;
  st.blob = blob, st.off_tokens = off_tokens, st.T = T;
  st.out_rows = reinterpret_cast<const int32_t *>(blob + off_rows);
  return run_conv_norm(st, a, EmbedPairs(), R, s);
}

}  // namespace ffmi
