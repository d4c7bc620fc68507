// residual.hip -- the 32-bit residual stream (residual.h): input rows, sums of
// sublayer outputs, norms.
#include "residual.h"

#include <algorithm>

#include "device_util.h"

namespace ffmi {

__global__ __launch_bounds__(256) void embed_pos_kernel(
    const char *__restrict__ blob_src, uint4 *__restrict__ blob_dst, int blob_n16,
    const uint16_t *__restrict__ embed, const uint16_t *__restrict__ pos, float *__restrict__ x,
    uint16_t *__restrict__ xb, int H) {
  const int t = blockIdx.x;
  const PagedToken tk = reinterpret_cast<const PagedToken *>(blob_src)[t];  // tokens come first
  const uint4 *src = reinterpret_cast<const uint4 *>(blob_src);
  for (int i = t * 256 + threadIdx.x; i < blob_n16; i += gridDim.x * 256) blob_dst[i] = src[i];
  for (int c = threadIdx.x; c < H / 8; c += 256) {
    f4 a, b, pa, pb;
    unpack8_bf16(*reinterpret_cast<const uint4 *>(embed + (size_t)tk.token * H + c * 8), a, b);
    if (pos) {
      unpack8_bf16(*reinterpret_cast<const uint4 *>(pos + (size_t)tk.pos * H + c * 8), pa, pb);
      a += pa, b += pb;
    }
    *reinterpret_cast<f4 *>(x + (size_t)t * H + c * 8) = a;
    *reinterpret_cast<f4 *>(x + (size_t)t * H + c * 8 + 4) = b;
    if (xb) *reinterpret_cast<uint4 *>(xb + act_packed_off(t, c * 8, H)) = pack8_bf16(a, b);
  }
}

hipError_t launch_embed_pos(const char *blob_src, char *blob_dst, size_t blob_bytes,
                            const uint16_t *embed, const uint16_t *pos, float *x, uint16_t *xb,
                            int T, int H, hipStream_t s) {
  if (T <= 0) return hipSuccess;
  if (H % 32) return hipErrorInvalidValue;
  hipLaunchKernelGGL(embed_pos_kernel, dim3(T), dim3(256), 0, s, blob_src,
                     reinterpret_cast<uint4 *>(blob_dst), (int)((blob_bytes + 15) / 16), embed, pos,
                     x, xb, H);
  return hipGetLastError();
}

// One workgroup per row; the slab, x and w loads of a chunk are all issued
// before the reduction.
//   PRE == false: x += y / rms(y) * w, hb the new x
//   PRE == true:  x += y, h = x / rms(x) * w to hb or hf (w null: the sum only);
//   without slabs x is, where em.table is given, an embedding row
struct EmbedRows {
  const char *blob_src = nullptr;  // staging, tokens first; copied to blob_dst
  uint4 *blob_dst = nullptr;
  int blob_n16 = 0;
  const uint16_t *table = nullptr;
  float scale = 1.f;
};
template <int NT, int MAXC, int MAXS, bool PRE>
__global__ __launch_bounds__(NT) void stream_norm_kernel(const float *__restrict__ yp, int S, int NP,
                                                         const float *__restrict__ w,
                                                         float *__restrict__ x,
                                                         uint16_t *__restrict__ hb,
                                                         float *__restrict__ hf, int H, int n,
                                                         float eps, EmbedRows em) {
  __shared__ float sh[NT / 64];
  const int row = blockIdx.x, T = gridDim.x, nchunk = H >> 3;
  const uint16_t *er = nullptr;
  if (PRE && MAXS == 0 && em.table) {
    er = em.table + (size_t)reinterpret_cast<const PagedToken *>(em.blob_src)[row].token * H;
    const uint4 *src = reinterpret_cast<const uint4 *>(em.blob_src);
    for (int i = row * NT + threadIdx.x; i < em.blob_n16; i += T * NT) em.blob_dst[i] = src[i];
  }
  f4 y[MAXC][2], xv[MAXC][2], wv[MAXC][2];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int ch = min((int)threadIdx.x + c * NT, nchunk - 1);
    f4 lo[MAXS ? MAXS : 1], hi[MAXS ? MAXS : 1];
    lo[0] = hi[0] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int sl = 0; sl < MAXS; ++sl) {
      const float *qs = yp + (size_t)row * NP + ch * 8 + (size_t)min(sl, S - 1) * T * NP;
      lo[sl] = *reinterpret_cast<const f4 *>(qs);
      hi[sl] = *reinterpret_cast<const f4 *>(qs + 4);
    }
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      if (!er) xv[c][h] = *reinterpret_cast<const f4 *>(x + (size_t)row * H + ch * 8 + 4 * h);
      wv[c][h] = f4{0.f, 0.f, 0.f, 0.f};
      if (!PRE || w) wv[c][h] = *reinterpret_cast<const f4 *>(w + ch * 8 + 4 * h);
    }
    if (er) {
      unpack8_bf16(*reinterpret_cast<const uint4 *>(er + ch * 8), xv[c][0], xv[c][1]);
      xv[c][0] *= em.scale, xv[c][1] *= em.scale;
    }
    y[c][0] = lo[0], y[c][1] = hi[0];
#pragma unroll
    for (int sl = 1; sl < MAXS; ++sl)
      if (sl < S) y[c][0] += lo[sl], y[c][1] += hi[sl];
    if constexpr (PRE) {
#pragma unroll
      for (int h = 0; h < 2; ++h) y[c][h] = xv[c][h] += y[c][h];
    }
    if ((int)threadIdx.x + c * NT < nchunk)
#pragma unroll
      for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int e = 0; e < 4; ++e) ss = fmaf(y[c][h][e], y[c][h][e], ss);
  }
  const float r = inv_rms(row_sum<NT>(ss, sh), n, eps);
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int ch = threadIdx.x + c * NT;
    if (ch >= nchunk) continue;
#pragma unroll
    for (int h = 0; h < 2; ++h)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float v = y[c][h][e] * r * wv[c][h][e];
        if constexpr (PRE) y[c][h][e] = v;
        else y[c][h][e] = xv[c][h][e] += v;
      }
    if (!PRE || MAXS || er) {
      *reinterpret_cast<f4 *>(x + (size_t)row * H + ch * 8) = xv[c][0];
      *reinterpret_cast<f4 *>(x + (size_t)row * H + ch * 8 + 4) = xv[c][1];
    }
    if (PRE && !w) continue;
    if (hb)
      *reinterpret_cast<uint4 *>(hb + act_packed_off(row, ch * 8, H)) = pack8_bf16(y[c][0], y[c][1]);
    if (PRE && hf) {
      *reinterpret_cast<f4 *>(hf + (size_t)row * H + ch * 8) = y[c][0];
      *reinterpret_cast<f4 *>(hf + (size_t)row * H + ch * 8 + 4) = y[c][1];
    }
  }
}

template <bool PRE>
static hipError_t run_stream_norm(Partials y, const float *w, float *x, uint16_t *hb, float *hf,
                                  int T, int H, int n, float eps, hipStream_t s,
                                  const EmbedRows &em = EmbedRows()) {
  if (T <= 0) return hipSuccess;
  if (H % 32 || y.S < (PRE ? 0 : 1) || y.S > 8) return hipErrorInvalidValue;
  if (y.S > 0 && (y.NP < H || y.NP % 4 || !y.p)) return hipErrorInvalidValue;
  const int nchunk = H / 8;
#define FFMI_SN(NT, MC, MS)                                                                       \
  hipLaunchKernelGGL((stream_norm_kernel<NT, MC, MS, PRE>), dim3(T), dim3(NT), 0, s, y.p, y.S, \
                     y.NP, w, x, hb, hf, H, n, eps, em)
#define FFMI_SNS(NT, MC)                   \
  do {                                     \
    if (PRE && y.S == 0) FFMI_SN(NT, MC, (PRE ? 0 : 1)); \
    else if (y.S == 1) FFMI_SN(NT, MC, 1); \
    else if (y.S == 2) FFMI_SN(NT, MC, 2); \
    else if (y.S <= 4) FFMI_SN(NT, MC, 4); \
    else FFMI_SN(NT, MC, 8);               \
  } while (0)
  if (nchunk <= 128) FFMI_SNS(128, 1);
  else if (nchunk <= 256) FFMI_SNS(256, 1);
  else if (nchunk <= 512) FFMI_SNS(512, 1);
  else if (nchunk <= 1024) FFMI_SNS(1024, 1);
  else if (nchunk <= 2048) FFMI_SNS(1024, 2);
  else return hipErrorInvalidValue;
#undef FFMI_SNS
#undef FFMI_SN
  return hipGetLastError();
}
hipError_t launch_post_norm(Partials y, const float *w, float *x, uint16_t *xb, int T, int H, int n,
                            float eps, hipStream_t s) {
  return run_stream_norm<false>(y, w, x, xb, nullptr, T, H, n, eps, s);
}
hipError_t launch_embed_norm(const char *blob_src, char *blob_dst, size_t blob_bytes,
                             const uint16_t *embed, float scale, const float *w, float *x,
                             uint16_t *hb, float *hf, int T, int H, int n, float eps, hipStream_t s) {
  EmbedRows em;
  em.blob_src = blob_src, em.blob_dst = reinterpret_cast<uint4 *>(blob_dst);
  em.blob_n16 = (int)((blob_bytes + 15) / 16), em.table = embed, em.scale = scale;
  return run_stream_norm<true>(Partials(), w, x, hb, hf, T, H, n, eps, s, em);
}
hipError_t launch_add_norm(Partials y, const float *w, float *x, uint16_t *hb, float *hf, int T,
                           int H, int n, float eps, hipStream_t s) {
  return run_stream_norm<true>(y, w, x, hb, hf, T, H, n, eps, s);
}

__global__ __launch_bounds__(256) void row_norm_kernel(const int32_t *__restrict__ rows,
                                                       const float *__restrict__ x,
                                                       const float *__restrict__ w,
                                                       uint16_t *__restrict__ hb,
                                                       float *__restrict__ hf, int H, int n,
                                                       float eps) {
  __shared__ float sh[4];
  const int i = blockIdx.x;
  const float *xr = x + (size_t)rows[i] * H;
  float ss = 0.f;
  for (int c = threadIdx.x; c < H / 4; c += 256) {
    const f4 v = *reinterpret_cast<const f4 *>(xr + c * 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) ss = fmaf(v[e], v[e], ss);
  }
  const float r = inv_rms(row_sum<256>(ss, sh), n, eps);
  for (int c = threadIdx.x; c < H / 8; c += 256) {
    f4 v[2];
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      v[h] = *reinterpret_cast<const f4 *>(xr + c * 8 + 4 * h);
      const f4 wv = *reinterpret_cast<const f4 *>(w + c * 8 + 4 * h);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[h][e] = v[h][e] * r * wv[e];
      if (hf) *reinterpret_cast<f4 *>(hf + (size_t)i * H + c * 8 + 4 * h) = v[h];
    }
    if (hb) *reinterpret_cast<uint4 *>(hb + act_packed_off(i, c * 8, H)) = pack8_bf16(v[0], v[1]);
  }
}

hipError_t launch_row_norm(const char *blob, int off_rows, const float *x, const float *w,
                           uint16_t *hb, float *hf, int R, int H, int n, float eps, hipStream_t s) {
  if (R <= 0) return hipSuccess;
  if (H % 32) return hipErrorInvalidValue;
  hipLaunchKernelGGL(row_norm_kernel, dim3(R), dim3(256), 0, s,
                     reinterpret_cast<const int32_t *>(blob + off_rows), x, w, hb, hf, H, n, eps);
  return hipGetLastError();
}

// One workgroup per row, a thread's chunks of 8 columns; all loads before the
// reduction, of slabs MAXS at a time.
template <int NT, int MAXC, int MAXS>
__global__ __launch_bounds__(NT) void sum_norm_kernel(SumNorm a) {
  constexpr int U = 4;  // expert rows in flight
  __shared__ float sh[NT / 64];
  const int row = blockIdx.x, H = a.H, nchunk = H >> 3;
  f4 x[MAXC][2], wv[MAXC][2];
  float ss = 0.f;
  const float alpha = a.own ? a.alpha + a.own[row] : a.alpha;
  const int32_t *at = a.rows ? a.at + (size_t)row * a.top : nullptr;
  const float *wt = a.rows ? a.wt + (size_t)row * a.top : nullptr;
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int ch = min((int)threadIdx.x + c * NT, nchunk - 1);
    f4 p[MAXS ? MAXS : 1][2];
    auto slabs = [&](int s0) {
#pragma unroll
      for (int sl = 0; sl < MAXS; ++sl) {
        const float *q = a.y.p + (size_t)row * a.y.NP + ch * 8 + (size_t)min(s0 + sl, a.y.S - 1) * a.T * a.y.NP;
        p[sl][0] = *reinterpret_cast<const f4 *>(q), p[sl][1] = *reinterpret_cast<const f4 *>(q + 4);
      }
    };
    slabs(0);
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      x[c][h] = *reinterpret_cast<const f4 *>(a.x + (size_t)row * H + ch * 8 + 4 * h) * alpha;
      wv[c][h] = *reinterpret_cast<const f4 *>(a.w + ch * 8 + 4 * h);
    }
    f4 y[2];
    y[0] = y[1] = f4{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; at && k0 < a.top; k0 += U) {
      f4 r[U][2];
      float w[U];
#pragma unroll
      for (int k = 0; k < U; ++k) {
        const int kk = min(k0 + k, a.top - 1), slot = at[kk];
        w[k] = k0 + k < a.top && slot >= 0 ? wt[kk] : 0.f;
        const size_t o = (size_t)max(slot, 0) * H + ch * 8;
        if (a.rows_f32) {
          const float *q = (const float *)a.rows + o;
          r[k][0] = *reinterpret_cast<const f4 *>(q), r[k][1] = *reinterpret_cast<const f4 *>(q + 4);
        } else {
          unpack8_bf16(*reinterpret_cast<const uint4 *>((const uint16_t *)a.rows + o), r[k][0], r[k][1]);
        }
      }
#pragma unroll
      for (int k = 0; k < U; ++k)
        if (w[k] != 0.f) y[0] += r[k][0] * w[k], y[1] += r[k][1] * w[k];
    }
    for (int s0 = 0; MAXS > 0 && s0 < a.y.S; s0 += MAXS ? MAXS : 1) {
      if (s0 > 0) slabs(s0);
#pragma unroll
      for (int sl = 0; sl < MAXS; ++sl)
        if (s0 + sl < a.y.S) y[0] += p[sl][0], y[1] += p[sl][1];
    }
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      x[c][h] += y[h];
      if ((int)threadIdx.x + c * NT < nchunk)
#pragma unroll
        for (int e = 0; e < 4; ++e) ss = fmaf(x[c][h][e], x[c][h][e], ss);
    }
  }
  const float r = inv_rms(row_sum<NT>(ss, sh), a.n, a.eps);
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int ch = threadIdx.x + c * NT;
    if (ch >= nchunk) continue;
#pragma unroll
    for (int h = 0; h < 2; ++h) {
#pragma unroll
      for (int e = 0; e < 4; ++e) x[c][h][e] = x[c][h][e] * r * wv[c][h][e];
      *reinterpret_cast<f4 *>(a.x + (size_t)row * H + ch * 8 + 4 * h) = x[c][h];
    }
    const uint4 b = pack8_bf16(x[c][0], x[c][1]);
    if (a.hb) *reinterpret_cast<uint4 *>(a.hb + act_packed_off(row, ch * 8, H)) = b;
    if (a.hrow) *reinterpret_cast<uint4 *>(a.hrow + (size_t)row * H + ch * 8) = b;
  }
}
hipError_t launch_sum_norm(const SumNorm &a, hipStream_t s) {
  if (a.T <= 0) return hipSuccess;
  if (a.H % 32 || !a.x || !a.w || a.y.S < 0 || a.y.S > 8 || (a.y.S > 0 && (a.y.NP < a.H || a.y.NP % 4)) ||
      (a.rows && (a.top < 1 || !a.at || !a.wt)))
    return hipErrorInvalidValue;
  const int nchunk = a.H / 8;
#define FFMI_SM(NT, MC, MS) hipLaunchKernelGGL((sum_norm_kernel<NT, MC, MS>), dim3(a.T), dim3(NT), 0, s, a)
#define FFMI_SMS(NT, MC)                 \
  do {                                   \
    if (a.y.S == 0) FFMI_SM(NT, MC, 0);  \
    else if (a.y.S == 1) FFMI_SM(NT, MC, 1); \
    else FFMI_SM(NT, MC, 4);             \
  } while (0)
  if (nchunk <= 128) FFMI_SMS(128, 1);
  else if (nchunk <= 256) FFMI_SMS(256, 1);
  else if (nchunk <= 512) FFMI_SMS(512, 1);
  else if (nchunk <= 1024) FFMI_SMS(1024, 1);
  else if (nchunk <= 2048) FFMI_SMS(1024, 2);
  else return hipErrorInvalidValue;
#undef FFMI_SMS
#undef FFMI_SM
  return hipGetLastError();
}

__global__ __launch_bounds__(256) void pack_sums_kernel(Partials y, int col, uint16_t *__restrict__ out, int T,
                                                        int n) {
  const int n8 = n >> 3;
  const long id = blockIdx.x * 256L + threadIdx.x;
  if (id >= (long)T * n8) return;
  const int t = (int)(id / n8), c = (int)(id % n8) * 8;
  const float *p = y.p + (size_t)t * y.NP + col + c;
  f4 lo = *reinterpret_cast<const f4 *>(p), hi = *reinterpret_cast<const f4 *>(p + 4);
  for (int s = 1; s < y.S; ++s) {
    const float *ps = p + (size_t)s * T * y.NP;
    lo += *reinterpret_cast<const f4 *>(ps), hi += *reinterpret_cast<const f4 *>(ps + 4);
  }
  *reinterpret_cast<uint4 *>(out + act_packed_off(t, c, n)) = pack8_bf16(lo, hi);
}
hipError_t launch_pack_sums(const Partials &y, int col, uint16_t *out, int T, int n, hipStream_t s) {
  if (T <= 0) return hipSuccess;
  if (n <= 0 || n % 32 || col % 4 || y.NP % 4 || y.S < 1 || col + n > y.NP) return hipErrorInvalidValue;
  hipLaunchKernelGGL(pack_sums_kernel, dim3((unsigned)(((long)T * (n / 8) + 255) / 256)), dim3(256), 0, s, y, col,
                     out, T, n);
  return hipGetLastError();
}

__global__ void relu2_f32_kernel(float *u, size_t n) {
  for (size_t i = blockIdx.x * (size_t)blockDim.x + threadIdx.x; i < n;
       i += (size_t)gridDim.x * blockDim.x) {
    const float v = fmaxf(u[i], 0.f);
    u[i] = v * v;
  }
}
hipError_t launch_relu2_f32(float *u, size_t n, hipStream_t s) {
  if (n == 0) return hipSuccess;
  hipLaunchKernelGGL(relu2_f32_kernel, dim3((unsigned)std::min<size_t>((n + 255) / 256, 16384)),
                     dim3(256), 0, s, u, n);
  return hipGetLastError();
}

__global__ void glu_f32_kernel(const float *__restrict__ gu, float *__restrict__ Y, int F, size_t n,
                               float limit) {
  for (size_t i = blockIdx.x * (size_t)blockDim.x + threadIdx.x; i < n;
       i += (size_t)gridDim.x * blockDim.x) {
    const size_t t = i / F, c = i % F;
    Y[i] = clamped_glu(gu[t * 2 * F + c], gu[t * 2 * F + F + c], limit);
  }
}
hipError_t launch_glu_f32(const float *gu, float *Y, int T, int F, float limit, hipStream_t s) {
  const size_t n = (size_t)T * F;
  if (n == 0) return hipSuccess;
  hipLaunchKernelGGL(glu_f32_kernel, dim3((unsigned)std::min<size_t>((n + 255) / 256, 16384)),
                     dim3(256), 0, s, gu, Y, F, n, limit);
  return hipGetLastError();
}

__global__ void swiglu_f32_kernel(const float *__restrict__ gu, float *__restrict__ Y, int F, size_t n, int ldy) {
  for (size_t i = blockIdx.x * (size_t)blockDim.x + threadIdx.x; i < n;
       i += (size_t)gridDim.x * blockDim.x) {
    const size_t t = i / F, c = i % F;
    Y[t * ldy + c] = silu_glu(gu[t * 2 * F + c], gu[t * 2 * F + F + c]);
  }
}
hipError_t launch_swiglu_f32(const float *gu, float *Y, int T, int F, int ldy, hipStream_t s) {
  const size_t n = (size_t)T * F;
  if (n == 0) return hipSuccess;
  hipLaunchKernelGGL(swiglu_f32_kernel, dim3((unsigned)std::min<size_t>((n + 255) / 256, 16384)),
                     dim3(256), 0, s, gu, Y, F, n, ldy);
  return hipGetLastError();
}

__global__ void soft_cap_kernel(float *z, int n, int ld, float cap) {
  float *row = z + (size_t)blockIdx.y * ld;
  for (int c = blockIdx.x * 256 + threadIdx.x; c < n; c += gridDim.x * 256) row[c] = cap * tanhf(__fdiv_rn(row[c], cap));
}
hipError_t launch_soft_cap(float *z, int R, int n, int ld, float cap, hipStream_t s) {
  if (R <= 0) return hipSuccess;
  if (!(cap > 0.f)) return hipErrorInvalidValue;
  hipLaunchKernelGGL(soft_cap_kernel, dim3(std::min((n + 255) / 256, 64), R), dim3(256), 0, s, z, n, ld, cap);
  return hipGetLastError();
}

}  // namespace ffmi
