// latent.hip -- latent attention over a paged cache (latent.h).
#include <algorithm>

#include "device_util.h"
#include "latent.h"

namespace ffmi {

// ---------------------------------------------------------------------------
// latent store: one wave per token
// ---------------------------------------------------------------------------
template <class E>
__device__ __forceinline__ void latent_store_token(const PagedToken &tk, const E *d, const float *w,
                                                   E *cache, int rank, int n, float eps) {
  const int lane = threadIdx.x & 63;
  float ss = 0.f;
  for (int i = lane; i < rank; i += 64) {
    const float v = ld_elem(d + i);
    ss = fmaf(v, v, ss);
  }
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) ss += __shfl_xor(ss, o);
  const float r = inv_rms(ss, n, eps);
  E *dst = cache + (size_t)tk.row * rank;
  for (int i = lane; i < rank; i += 64) st_elem(dst + i, ld_elem(d + i) * r * w[i]);
}

__global__ __launch_bounds__(256) void latent_store_f32_kernel(const PagedToken *__restrict__ tok,
                                                               int T, LatentStore st) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t >= T) return;
  latent_store_token(tok[t], (const float *)st.d + (size_t)t * st.ldd, st.w, (float *)st.cache,
                     st.rank, st.n, st.eps);
}
hipError_t launch_latent_store_f32(const char *blob, int off_tokens, int T, const LatentStore &st,
                                   hipStream_t s) {
  if (T <= 0) return hipSuccess;
  hipLaunchKernelGGL(latent_store_f32_kernel, dim3((T + 3) / 4), dim3(256), 0, s,
                     reinterpret_cast<const PagedToken *>(blob + off_tokens), T, st);
  return hipGetLastError();
}

// ---------------------------------------------------------------------------
// per-head products (bf16 MFMA): Y[t][h][n] = sum_k X[t][h][k] W_h[n][k]
// ---------------------------------------------------------------------------
// W_h tile-major: block (h, nt, kt) of 16 x 32 at ((h * NTt + nt) * KT + kt) *
// 512.  Four waves, WM of them over row groups of MT tiles, 4 / WM over groups
// of NT weight tiles.  D = W . X^T: a lane holds four consecutive columns of
// one row.
struct HgDev {
  const uint16_t *X, *W, *gate;
  uint16_t *Y;
  int T, heads, KT, NTt, ldx, ldg, packed;
  int gx, gz;  // weight-tile groups, row groups of the launch
};
template <int MT, int NT, int WM>
__device__ __forceinline__ void head_gemm_block(const HgDev &a, int b) {
  constexpr int WN = 4 / WM;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4, l15 = lane & 15;
  const int bx = b % a.gx, h = (b / a.gx) % a.heads, bz = b / (a.gx * a.heads);
  const int nt0 = (bx * WN + wave % WN) * NT;
  const int m0 = (bz * WM + wave / WN) * MT * 16;
  if (nt0 >= a.NTt || m0 >= a.T) return;
  const int K = a.KT * 32;
  const uint16_t *xr[MT], *wr[NT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
    xr[i] = a.X + (size_t)min(m0 + i * 16 + l15, a.T - 1) * a.ldx + (size_t)h * K + 8 * g;
#pragma unroll
  for (int j = 0; j < NT; ++j)
    wr[j] = a.W + ((size_t)h * a.NTt + min(nt0 + j, a.NTt - 1)) * a.KT * 512 + lane * 8;
  f4 acc[MT][NT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[i][j] = f4{0.f, 0.f, 0.f, 0.f};
  constexpr int U = MT * NT >= 8 ? 2 : 4;  // k-steps of loads issued ahead of their MFMAs
  for (int k0 = 0; k0 < a.KT; k0 += U) {
    bf8 x[U][MT], w[U][NT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = min(k0 + u, a.KT - 1);
#pragma unroll
      for (int j = 0; j < NT; ++j) w[u][j] = *reinterpret_cast<const bf8 *>(wr[j] + (size_t)k * 512);
#pragma unroll
      for (int i = 0; i < MT; ++i) x[u][i] = *reinterpret_cast<const bf8 *>(xr[i] + k * 32);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (k0 + u < a.KT)
#pragma unroll
        for (int i = 0; i < MT; ++i)
#pragma unroll
          for (int j = 0; j < NT; ++j)
            acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[u][j], x[u][i], acc[i][j], 0, 0, 0);
  }
  const int N = a.NTt * 16, Yw = a.heads * N;
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const int m = m0 + i * 16 + l15;
    if (m >= a.T) continue;
    float sc = 1.f;
    if (a.gate) sc = __fdiv_rn(1.0f, 1.0f + expf(-bf2f(a.gate[(size_t)m * a.ldg + h])));
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      if (nt0 + j >= a.NTt) continue;
      const int n = h * N + (nt0 + j) * 16 + 4 * g;
      const f4 v = acc[i][j];
      const uint2 o = make_uint2(f2bf(v[0] * sc) | ((uint32_t)f2bf(v[1] * sc) << 16),
                                 f2bf(v[2] * sc) | ((uint32_t)f2bf(v[3] * sc) << 16));
      *reinterpret_cast<uint2 *>(a.Y + (a.packed ? act_packed_off(m, n, Yw) : (size_t)m * Yw + n)) = o;
    }
  }
}

template <int MT, int NT, int WM>
__global__ __launch_bounds__(256) void latent_prep_kernel(const PagedToken *__restrict__ tok,
                                                          HgDev a, int nprod, LatentStore st) {
  if ((int)blockIdx.x < nprod) {
    head_gemm_block<MT, NT, WM>(a, blockIdx.x);
    return;
  }
  const int t = (blockIdx.x - nprod) * 4 + (threadIdx.x >> 6);
  if (t >= a.T) return;
  latent_store_token(tok[t], (const uint16_t *)st.d + (size_t)t * st.ldd, st.w,
                     (uint16_t *)st.cache, st.rank, st.n, st.eps);
}

static hipError_t run_prep(const PagedToken *tok, const LatentStore &st, const HeadGemm &hg,
                           hipStream_t s) {
  if (hg.T <= 0) return hipSuccess;
  if (hg.K % 32 || hg.N % 32 || hg.ldx % 8) return hipErrorInvalidValue;
  HgDev a;
  a.X = (const uint16_t *)hg.X, a.W = (const uint16_t *)hg.W, a.gate = (const uint16_t *)hg.gate;
  a.Y = (uint16_t *)hg.Y;
  a.T = hg.T, a.heads = hg.heads, a.KT = hg.K / 32, a.NTt = hg.N / 16, a.ldx = hg.ldx;
  a.ldg = hg.ldg, a.packed = hg.packed ? 1 : 0;
  const int nst = st.cache ? (hg.T + 3) / 4 : 0;
#define FFMI_PREP(MT, NT, WM)                                                                   \
  do {                                                                                          \
    a.gx = (a.NTt + (4 / WM) * NT - 1) / ((4 / WM) * NT);                                       \
    a.gz = (hg.T + WM * MT * 16 - 1) / (WM * MT * 16);                                          \
    const int np = a.gx * a.heads * a.gz;                                                       \
    hipLaunchKernelGGL((latent_prep_kernel<MT, NT, WM>), dim3(np + nst), dim3(256), 0, s, tok, a, \
                       np, st);                                                                 \
  } while (0)
  if (hg.T <= 16) FFMI_PREP(1, 1, 1);
  else if (hg.T <= 32) FFMI_PREP(2, 1, 1);
  else if (hg.T <= 128) FFMI_PREP(2, 2, 1);
  else FFMI_PREP(4, 4, 2);
#undef FFMI_PREP
  return hipGetLastError();
}
hipError_t launch_latent_prep(const char *blob, int off_tokens, const LatentStore &st,
                              const HeadGemm &hg, hipStream_t s) {
  return run_prep(reinterpret_cast<const PagedToken *>(blob + off_tokens), st, hg, s);
}
hipError_t launch_head_gemm(const HeadGemm &hg, hipStream_t s) {
  return run_prep(nullptr, LatentStore(), hg, s);
}

// fp32: W_h as [K][N] row-major, one workgroup per (token, head)
__global__ __launch_bounds__(256) void head_gemm_f32_kernel(const float *__restrict__ X,
                                                            const float *__restrict__ W,
                                                            const float *__restrict__ gate,
                                                            float *__restrict__ Y, int heads, int K,
                                                            int N, int ldx, int ldg) {
  const int t = blockIdx.x, h = blockIdx.y;
  const float *x = X + (size_t)t * ldx + (size_t)h * K, *w = W + (size_t)h * K * N;
  const float sc =
      gate ? __fdiv_rn(1.0f, 1.0f + expf(-gate[(size_t)t * ldg + h])) : 1.0f;
  for (int n = threadIdx.x; n < N; n += 256) {
    float acc = 0.f;
    for (int k = 0; k < K; ++k) acc = fmaf(x[k], w[(size_t)k * N + n], acc);
    Y[((size_t)t * heads + h) * N + n] = acc * sc;
  }
}
hipError_t launch_head_gemm_f32(const HeadGemm &hg, hipStream_t s) {
  if (hg.T <= 0) return hipSuccess;
  hipLaunchKernelGGL(head_gemm_f32_kernel, dim3(hg.T, hg.heads), dim3(256), 0, s,
                     (const float *)hg.X, (const float *)hg.W, (const float *)hg.gate,
                     (float *)hg.Y, hg.heads, hg.K, hg.N, hg.ldx, hg.ldg);
  return hipGetLastError();
}

// ---------------------------------------------------------------------------
// attention over the pages, MFMA form
// ---------------------------------------------------------------------------
// One workgroup of eight waves: up to RT * 16 rows against a range of 64-token
// pages.  Scores S^T = C . Q'^T (lane: 4 keys of one row), outputs O^T = C^T .
// P^T with C^T read from the row-major page in LDS by the transposing LDS load;
// the k order of the second product is the key order the scores already have
// in the lanes (16-lane group g: keys 4g..4g+3 and 16+4g..).
//   scores:  wave = (16-key tile, half of the rows); RT == 1: four waves only
//   outputs: each wave an eighth of the latent's columns, all rows
// Softmax state in fp32, base-2 exponents; weights meet the second product in
// bf16, the sums take them unrounded.
typedef short s4 __attribute__((ext_vector_type(4)));
typedef short s8 __attribute__((ext_vector_type(8)));
typedef uint32_t u4 __attribute__((ext_vector_type(4)));
constexpr int kRankPad = 8;  // LDS row padding (elements)

template <int RC, int RT>
__global__ __launch_bounds__(512) void latent_attn_kernel(
    const char *__restrict__ blob, int off_blocks, const uint16_t *__restrict__ Q,
    const uint16_t *__restrict__ cache, uint16_t *__restrict__ O, float *__restrict__ slabs,
    float *__restrict__ ml, int heads, float scale_log2) {
  constexpr int R = RC * 64, KS = RC * 2, LDC = R + kRankPad;
  constexpr int SR = RT == 4 ? 2 : 1;           // row tiles of a wave's scores
  constexpr int NT = RC * 4, DT = (NT + 7) / 8;  // column tiles: all, of a wave's outputs
  constexpr int LDP = kPageTokens + 8;
  __shared__ __attribute__((aligned(16))) uint16_t sC[2][64 * LDC];
  __shared__ __attribute__((aligned(16))) uint16_t sP[RT * 16 * LDP];
  __shared__ float sM[4][RT * 16], sL[4][RT * 16];
  const PagedBlock bk = reinterpret_cast<const PagedBlock *>(blob + off_blocks)[blockIdx.x];
  if (bk.nrows <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, l15 = lane & 15;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int wk = wave & 3, wr = wave >> 2;
  const bool scoring = RT > 1 || wr == 0;
  const int32_t *table = reinterpret_cast<const int32_t *>(blob) + bk.table;

  // the next page: through registers, RC 16-byte chunks per thread, or (R ==
  // 512: a row is one 1 KiB wave access) straight into LDS where those
  // registers would not fit
  constexpr bool DMA = RC == 8 && RT == 4;
  auto page_at = [&](int i0) {
    return cache + (size_t)(i0 == 0 ? bk.page0 : table[bk.tile0 + i0]) * (64 * R);
  };
  auto dma = [&](int i0, int buf) {
    const uint16_t *page = page_at(i0);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int row = wave * 8 + i;
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) void *)(page + (size_t)row * R + lane * 8),
          (__attribute__((address_space(3))) void *)(&sC[buf][row * LDC]), 16, 0, 0);
    }
  };
  u4 pre[RC];
  auto fetch = [&](int i0) {
    const uint16_t *page = page_at(i0);
#pragma unroll
    for (int i = 0; i < RC; ++i) pre[i] = *reinterpret_cast<const u4 *>(page + (tid + i * 512) * 8);
  };
  auto stage = [&](int buf) {
#pragma unroll
    for (int i = 0; i < RC; ++i) {
      const int c = tid + i * 512;
      *reinterpret_cast<u4 *>(&sC[buf][(c / (R / 8)) * LDC + (c % (R / 8)) * 8]) = pre[i];
    }
  };
  if constexpr (DMA) dma(0, 0);
  else fetch(0);
  // this wave's rows of Q' as B operands (rows past the block re-read its last)
  bf8 q[SR][KS];
  int qpos[SR];
#pragma unroll
  for (int i = 0; i < SR; ++i) {
    const int r = min((wr * SR + i) * 16 + l15, bk.nrows - 1);
    const uint16_t *qr = Q + (size_t)(bk.row0 + r) * R + 8 * g;
#pragma unroll
    for (int k = 0; k < KS; ++k) q[i][k] = *reinterpret_cast<const bf8 *>(qr + k * 32);
    qpos[i] = bk.pos0 + (bk.row0 + r - bk.seg_row) / heads;
  }
  f4 acc[RT][DT];
#pragma unroll
  for (int i = 0; i < RT; ++i)
#pragma unroll
    for (int d = 0; d < DT; ++d) acc[i][d] = f4{0.f, 0.f, 0.f, 0.f};
  float m[RT], l[SR];
#pragma unroll
  for (int i = 0; i < RT; ++i) m[i] = -1e30f;
#pragma unroll
  for (int i = 0; i < SR; ++i) l[i] = 0.f;
  if constexpr (DMA) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  } else {
    stage(0);
    if (bk.ntiles > 1) fetch(1);
  }
  __syncthreads();
  for (int it = 0; it < bk.ntiles; ++it) {
    if constexpr (DMA)  // (its buffer was last read before the previous round's last barrier)
      if (it + 1 < bk.ntiles) dma(it + 1, (it + 1) & 1);
    const uint16_t *C = sC[it & 1];
    f4 s[SR];
    if (scoring) {
      // two chains per row tile (even / odd k-steps)
      f4 s2[SR];
#pragma unroll
      for (int i = 0; i < SR; ++i) s[i] = s2[i] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ks += 2) {
        const uint16_t *cr = &C[(wk * 16 + l15) * LDC + ks * 32 + 8 * g];
        const bf8 c0 = *reinterpret_cast<const bf8 *>(cr), c1 = *reinterpret_cast<const bf8 *>(cr + 32);
#pragma unroll
        for (int i = 0; i < SR; ++i) {
          s[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(c0, q[i][ks], s[i], 0, 0, 0);
          s2[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(c1, q[i][ks + 1], s2[i], 0, 0, 0);
        }
      }
      // scale, mask, this wave's maximum of every row
      const int key0 = (bk.tile0 + it) * 64 + wk * 16 + 4 * g;
#pragma unroll
      for (int i = 0; i < SR; ++i) {
        float mx = -1e30f;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float v = key0 + e <= qpos[i] ? (s[i][e] + s2[i][e]) * scale_log2 : -INFINITY;
          s[i][e] = v;
          mx = fmaxf(mx, v);
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16));
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        if (g == 0) sM[wk][(wr * SR + i) * 16 + l15] = mx;
      }
    }
    __syncthreads();
    float alpha[RT];
    bool moved = false;
#pragma unroll
    for (int i = 0; i < RT; ++i) {
      float mn = m[i];
#pragma unroll
      for (int k = 0; k < 4; ++k) mn = fmaxf(mn, sM[k][i * 16 + l15]);
      alpha[i] = __builtin_amdgcn_exp2f(m[i] - mn);
      moved |= mn != m[i];
      m[i] = mn;
    }
    if (scoring) {
#pragma unroll
      for (int i = 0; i < SR; ++i) {
        const float mi = RT > 1 && wr ? m[RT > 1 ? SR + i : i] : m[i];
        const float ai = RT > 1 && wr ? alpha[RT > 1 ? SR + i : i] : alpha[i];
        float p[4], sum = 0.f;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          p[e] = __builtin_amdgcn_exp2f(s[i][e] - mi);
          sum += p[e];
        }
        *reinterpret_cast<uint2 *>(&sP[((wr * SR + i) * 16 + l15) * LDP + wk * 16 + 4 * g]) =
            make_uint2(f2bf(p[0]) | ((uint32_t)f2bf(p[1]) << 16),
                       f2bf(p[2]) | ((uint32_t)f2bf(p[3]) << 16));
        l[i] = l[i] * ai + sum;
      }
    }
    if (!DMA && it + 1 < bk.ntiles) {
      stage((it + 1) & 1);  // (last read by the outputs of tile it - 1)
      if (it + 2 < bk.ntiles) fetch(it + 2);
    }
    __syncthreads();
    if (__any(moved))
#pragma unroll
      for (int i = 0; i < RT; ++i)
#pragma unroll
        for (int d = 0; d < DT; ++d) acc[i][d] *= alpha[i];
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      s8 p[RT];
#pragma unroll
      for (int i = 0; i < RT; ++i) {
        const uint16_t *pr = &sP[(i * 16 + l15) * LDP + kb * 32 + 4 * g];
        const s4 lo = *reinterpret_cast<const s4 *>(pr), hi = *reinterpret_cast<const s4 *>(pr + 16);
        p[i] = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
      }
#pragma unroll
      for (int d = 0; d < DT; ++d) {
        if (NT % 8 && wave * DT + d >= NT) continue;
        const uint16_t *cr =
            &C[(kb * 32 + 4 * g + (l15 >> 2)) * LDC + (wave * DT + d) * 16 + 4 * (l15 & 3)];
        const s4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (__attribute__((address_space(3))) s4 *)(cr));
        const s4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (__attribute__((address_space(3))) s4 *)(cr + 16 * LDC));
        const bf8 a = __builtin_bit_cast(
            bf8, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
#pragma unroll
        for (int i = 0; i < RT; ++i)
          acc[i][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, __builtin_bit_cast(bf8, p[i]),
                                                              acc[i][d], 0, 0, 0);
      }
    }
    if constexpr (DMA) {
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
      __syncthreads();
    }
  }
  if (scoring) {
#pragma unroll
    for (int i = 0; i < SR; ++i) {
      float v = l[i];
      v += __shfl_xor(v, 16);
      v += __shfl_xor(v, 32);
      if (g == 0) sL[wk][(wr * SR + i) * 16 + l15] = v;
    }
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < RT; ++i) {
    float sum = sL[0][i * 16 + l15];
#pragma unroll
    for (int k = 1; k < 4; ++k) sum += sL[k][i * 16 + l15];
    const int r = i * 16 + l15;
    if (r >= bk.nrows) continue;
    if (bk.slot >= 0) {
      const size_t pr = (size_t)bk.slot * (RT * 16) + r;
#pragma unroll
      for (int d = 0; d < DT; ++d)
        if (NT % 8 == 0 || wave * DT + d < NT)
          *reinterpret_cast<f4 *>(slabs + pr * R + (wave * DT + d) * 16 + 4 * g) = acc[i][d];
      if (wave == 0 && g == 0) ml[pr * 2] = m[i], ml[pr * 2 + 1] = sum;
    } else {
      const float inv = __fdiv_rn(1.0f, sum);
      uint16_t *o = O + (size_t)(bk.row0 + r) * R + wave * DT * 16 + 4 * g;
#pragma unroll
      for (int d = 0; d < DT; ++d) {
        if (NT % 8 && wave * DT + d >= NT) continue;
        const f4 v = acc[i][d] * inv;
        *reinterpret_cast<uint2 *>(o + d * 16) =
            make_uint2(f2bf(v[0]) | ((uint32_t)f2bf(v[1]) << 16),
                       f2bf(v[2]) | ((uint32_t)f2bf(v[3]) << 16));
      }
    }
  }
}

// partials of split blocks, in slot order: one workgroup per row, the slots'
// weights first (one lane each), then the slabs in groups of independent loads
template <int RC>
constexpr int kMergeThreads = RC <= 4 ? 64 : 128;
template <int RC>
__global__ __launch_bounds__(kMergeThreads<RC>) void latent_merge_kernel(
    const char *__restrict__ blob, int off_merges, const float *__restrict__ slabs,
    const float *__restrict__ ml, uint16_t *__restrict__ O, int block_rows) {
  constexpr int R = RC * 64, G = 8;
  const PagedMerge mg = reinterpret_cast<const PagedMerge *>(blob + off_merges)[blockIdx.x];
  const int r = blockIdx.y, lane = threadIdx.x & 63;
  if (r >= mg.nrows) return;
  const size_t row0 = (size_t)mg.slot0 * block_rows + r;
  const int col = threadIdx.x * 4;
  const float *sl = slabs + row0 * R + min(col, R - 4);
  f4 acc = f4{0.f, 0.f, 0.f, 0.f};
  float M = -1e30f, sum = 0.f;
  constexpr int L = 64;  // slots at a time (every wave works out the same weights)
  for (int s0 = 0; s0 < mg.nslots; s0 += L) {
    const int n = min(L, mg.nslots - s0);
    const size_t mi = (row0 + (size_t)(s0 + min(lane, n - 1)) * block_rows) * 2;
    const float m = lane < n ? ml[mi] : -1e30f, l = lane < n ? ml[mi + 1] : 0.f;
    float mx = m;
#pragma unroll
    for (int o = L / 2; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o));
    mx = fmaxf(mx, M);
    const float a = __builtin_amdgcn_exp2f(M - mx), w = __builtin_amdgcn_exp2f(m - mx);
    float ls = w * l;
#pragma unroll
    for (int o = L / 2; o > 0; o >>= 1) ls += __shfl_xor(ls, o);
    sum = sum * a + ls;
    acc *= a;
    M = mx;
    for (int i0 = 0; i0 < n; i0 += G) {
      f4 v[G];
#pragma unroll
      for (int i = 0; i < G; ++i)
        v[i] = *reinterpret_cast<const f4 *>(sl + (size_t)(s0 + min(i0 + i, n - 1)) * block_rows * R);
#pragma unroll
      for (int i = 0; i < G; ++i) {
        const float wi = i0 + i < n ? __shfl(w, i0 + i) : 0.f;
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[e] = fmaf(wi, v[i][e], acc[e]);
      }
    }
  }
  const float inv = __fdiv_rn(1.0f, sum);
  if (col >= R) return;
  *reinterpret_cast<uint2 *>(O + (size_t)(mg.row0 + r) * R + col) =
      make_uint2(f2bf(acc[0] * inv) | ((uint32_t)f2bf(acc[1] * inv) << 16),
                 f2bf(acc[2] * inv) | ((uint32_t)f2bf(acc[3] * inv) << 16));
}

bool latent_rank_supported(int rank) {
  const int rc = rank / 64;
  return rank % 64 == 0 && (rc == 1 || rc == 2 || rc == 3 || rc == 4 || rc == 6 || rc == 8);
}

hipError_t launch_latent_attention(const char *blob, const PagedLists &pl, const uint16_t *q,
                                   const uint16_t *cache, uint16_t *o, float *slabs, float *ml,
                                   int rank, float scale, hipStream_t s) {
  if (pl.num_blocks <= 0) return hipSuccess;
  const float sl = scale * 1.4426950408889634f;
#define FFMI_LA2(RC, RT)                                                                        \
  hipLaunchKernelGGL((latent_attn_kernel<RC, RT>), dim3(pl.num_blocks), dim3(512), 0, s, blob,  \
                     pl.off_blocks, q, cache, o, slabs, ml, pl.heads, sl)
#define FFMI_LA(RC)                                                                             \
  case RC:                                                                                      \
    if (pl.row_tiles == 1) FFMI_LA2(RC, 1);                                                     \
    else if (pl.row_tiles == 2) FFMI_LA2(RC, 2);                                                \
    else if (pl.row_tiles == 4) FFMI_LA2(RC, 4);                                                \
    else return hipErrorInvalidValue;                                                           \
    if (pl.num_merges > 0)                                                                      \
      hipLaunchKernelGGL((latent_merge_kernel<RC>), dim3(pl.num_merges, pl.row_tiles * 16),     \
                         dim3(kMergeThreads<RC>), 0, s, blob, pl.off_merges, slabs, ml, o,                \
                         pl.row_tiles * 16);                                                    \
    break
  if (rank % 64) return hipErrorInvalidValue;
  switch (rank / 64) {
    FFMI_LA(1);
    FFMI_LA(2);
    FFMI_LA(3);
    FFMI_LA(4);
    FFMI_LA(6);
    FFMI_LA(8);
    default: return hipErrorInvalidValue;
  }
#undef FFMI_LA
#undef FFMI_LA2
  return hipGetLastError();
}

// ---------------------------------------------------------------------------
// attention, one workgroup per row (fp32, and bf16 ranks without an MFMA form)
// ---------------------------------------------------------------------------
constexpr int kRowsMaxRank = 2048;
template <class E>
__global__ __launch_bounds__(256) void latent_rows_kernel(const char *__restrict__ blob,
                                                          int off_blocks, const E *__restrict__ Q,
                                                          const E *__restrict__ cache,
                                                          E *__restrict__ O, int heads, int rank,
                                                          float scale) {
  __shared__ float sq[kRowsMaxRank], sp[256], red[4];
  __shared__ int srow[256];
  const PagedBlock bk = reinterpret_cast<const PagedBlock *>(blob + off_blocks)[blockIdx.x];
  const int r = blockIdx.y, tid = threadIdx.x;
  if (r >= bk.nrows) return;
  const int32_t *table = reinterpret_cast<const int32_t *>(blob) + bk.table;
  const size_t row = (size_t)bk.row0 + r;
  const int n = bk.pos0 + (int)(row - bk.seg_row) / heads + 1;  // visible positions
  for (int i = tid; i < rank; i += 256) sq[i] = ld_elem(Q + row * rank + i);
  float acc[kRowsMaxRank / 256];
#pragma unroll
  for (int i = 0; i < kRowsMaxRank / 256; ++i) acc[i] = 0.f;
  float m = -1e30f, l = 0.f;
  for (int j0 = 0; j0 < n; j0 += 256) {
    __syncthreads();
    const int j = j0 + tid;
    float sv = -INFINITY;
    if (j < n) {
      const int cr = table[j >> 6] * kPageTokens + (j & 63);
      srow[tid] = cr;
      const E *c = cache + (size_t)cr * rank;
      float a = 0.f;
      for (int i = 0; i < rank; ++i) a = fmaf(sq[i], ld_elem(c + i), a);
      sv = a * scale;
    }
    float mx = sv;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o));
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    const float mn = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float p = j < n ? expf(sv - mn) : 0.f;
    sp[tid] = p;
    float sum = p;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) sum += __shfl_xor(sum, o);
    __syncthreads();
    if ((tid & 63) == 0) red[tid >> 6] = sum;
    __syncthreads();
    const float al = expf(m - mn);
    l = l * al + (red[0] + red[1] + red[2] + red[3]);
    m = mn;
    const int cnt = min(256, n - j0);
#pragma unroll
    for (int i = 0; i < kRowsMaxRank / 256; ++i) {
      const int d = tid + i * 256;
      if (d >= rank) break;
      float a = acc[i] * al;
      for (int k = 0; k < cnt; ++k) a = fmaf(sp[k], ld_elem(cache + (size_t)srow[k] * rank + d), a);
      acc[i] = a;
    }
  }
  const float inv = __fdiv_rn(1.0f, l);
#pragma unroll
  for (int i = 0; i < kRowsMaxRank / 256; ++i) {
    const int d = tid + i * 256;
    if (d < rank) st_elem(O + row * rank + d, acc[i] * inv);
  }
}

hipError_t launch_latent_attention_rows(const char *blob, const PagedLists &pl, const void *q,
                                        const void *cache, void *o, int rank, float scale,
                                        bool bf16, hipStream_t s) {
  if (pl.num_blocks <= 0) return hipSuccess;
  if (rank > kRowsMaxRank || pl.num_merges > 0) return hipErrorInvalidValue;
  const dim3 grid(pl.num_blocks, pl.row_tiles * 16);
  if (bf16)
    hipLaunchKernelGGL(latent_rows_kernel<uint16_t>, grid, dim3(256), 0, s, blob, pl.off_blocks,
                       (const uint16_t *)q, (const uint16_t *)cache, (uint16_t *)o, pl.heads, rank,
                       scale);
  else
    hipLaunchKernelGGL(latent_rows_kernel<float>, grid, dim3(256), 0, s, blob, pl.off_blocks,
                       (const float *)q, (const float *)cache, (float *)o, pl.heads, rank, scale);
  return hipGetLastError();
}

}  // namespace ffmi
