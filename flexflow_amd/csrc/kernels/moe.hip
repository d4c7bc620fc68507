// moe.hip -- mixture of experts (moe.h).
#include "moe.h"

#include <algorithm>

#include "device_util.h"

namespace ffmi {

// ---------------------------------------------------------------------------
// routing
// ---------------------------------------------------------------------------
// a column's sum over the slabs, their loads together
__device__ __forceinline__ float slab_total(const Partials &z, const float *p, size_t slab) {
  float v[8];
#pragma unroll
  for (int s = 0; s < 8; ++s) v[s] = p[min(s, z.S - 1) * slab];
#pragma unroll
  for (int s = 1; s < 8; ++s)
    if (s < z.S) v[0] += v[s];
  return v[0];
}
// the wave's largest value, NV a lane (column i * 64 + lane; the lowest among equals)
template <int NV>
__device__ __forceinline__ int best_column(const float (&v)[NV], float &best) {
  const int lane = threadIdx.x & 63;
  int at = lane;
  best = v[0];
#pragma unroll
  for (int i = 1; i < NV; ++i)
    if (v[i] > best) best = v[i], at = i * 64 + lane;
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float b = __shfl_xor(best, o);
    const int w = __shfl_xor(at, o);
    if (b > best || (b == best && w < at)) best = b, at = w;
  }
  return at;
}
// A wave picks a token's experts: NV logits a lane, the best of the wave `top`
// times over.
template <int NV>
__device__ __forceinline__ void pick_experts(const Partials &z, const float *__restrict__ bias, const MoeSizes &n,
                                             int t, const MoeLists &l) {
  const int lane = threadIdx.x & 63;
  const size_t slab = (size_t)n.T * z.NP;
  const float *row = z.p + (size_t)t * z.NP;
  const float gate = n.shared ? slab_total(z, row + n.gate_col, slab) : 0.f;
  float v[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int e = i * 64 + lane;
    v[i] = -INFINITY;
    if (e < n.experts) {
      v[i] = slab_total(z, row + e, slab) + bias[e];
    }
  }
  float top0 = 0.f, sum = 0.f, mine = 0.f;  // lane k: the k-th pick
  int mine_e = 0;
  for (int k = 0; k < n.top; ++k) {
    float best;
    const int at = best_column<NV>(v, best);
    if (k == 0) top0 = best;
    const float p = expf(best - top0);
    sum += p;
    if (lane == k) mine = p, mine_e = at;
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (at == i * 64 + lane) v[i] = -INFINITY;
  }
  if (lane < n.top) {
    l.picked[(size_t)t * n.top + lane] = min(mine_e, n.experts - 1);
    l.wt[(size_t)t * n.top + lane] = __fdiv_rn(mine, sum);
  }
  if (n.shared && lane == 0) l.gate[t] = __fdiv_rn(1.0f, 1.0f + expf(-gate));
}
// the same by scores
template <int NV>
__device__ __forceinline__ void pick_experts(const Partials &z, const MoeScores &sc, const MoeSizes &n, int t,
                                             const MoeLists &l) {
  const int lane = threadIdx.x & 63, cols = n.experts + n.identity, size = cols / sc.groups;
  const size_t slab = (size_t)n.T * z.NP;
  const float *row = z.p + (size_t)t * z.NP;
  float s[NV], v[NV];
  float mx = -INFINITY, sum = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int e = i * 64 + lane;
    s[i] = e < cols ? slab_total(z, row + e, slab) : -INFINITY;
    mx = fmaxf(mx, s[i]);
  }
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o));
#pragma unroll
  for (int i = 0; i < NV; ++i) s[i] = expf(s[i] - mx), sum += s[i];
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) sum += __shfl_xor(sum, o);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int e = i * 64 + lane;
    s[i] = __fdiv_rn(s[i], sum);
    v[i] = e < cols ? s[i] + sc.correction[e] : -INFINITY;
  }
  if (sc.keep < sc.groups) {  // the group of the best column left, `keep` times over
    float left[NV];
    bool in[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) left[i] = v[i], in[i] = false;
    for (int k = 0; k < sc.keep; ++k) {
      float best;
      const int g = best_column<NV>(left, best) / size;
#pragma unroll
      for (int i = 0; i < NV; ++i)
        if ((i * 64 + lane) / size == g) in[i] = true, left[i] = -INFINITY;
    }
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (!in[i]) v[i] = -INFINITY;
  }
  float mine = 0.f, total = 0.f, own = 0.f;
  int mine_e = 0;
  for (int k = 0; k < n.top; ++k) {
    float best, w = 0.f;
    const int at = best_column<NV>(v, best);
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (at == i * 64 + lane) v[i] = -INFINITY, w = s[i];
    w = __shfl(w, at & 63);
    total += w;
    if (at >= n.experts) own += w;
    if (lane == k) mine = w, mine_e = at;
  }
  const float f = __fdiv_rn(sc.scale, total + 1e-20f);
  if (lane < n.top) {
    const bool real = mine_e < n.experts;
    l.picked[(size_t)t * n.top + lane] = real ? mine_e : -1;
    l.wt[(size_t)t * n.top + lane] = real ? mine * f : 0.f;
  }
  if (n.identity && lane == 0) l.own[t] = own * f;
}
// How: `const float *` (bias) or MoeScores
template <int NV, class How>
__global__ __launch_bounds__(256) void moe_pick_kernel(Partials z, How how, MoeSizes n, MoeLists l) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t < n.T) pick_experts<NV>(z, how, n, t, l);
}

// One workgroup: tokens by expert.  PICK: it picks the experts as well (few tokens).
template <int NV, bool PICK, class How>
__global__ __launch_bounds__(1024) void moe_lists_kernel(Partials z, How how, MoeSizes n, MoeLists l,
                                                         int rows) {
  __shared__ int count[kMoeMaxExperts], next[kMoeMaxExperts], total;
  const int tid = threadIdx.x, A = n.T * n.top, st = n.shared_tiles(rows);
  for (int e = tid; e < n.experts; e += 1024) count[e] = 0;
  if constexpr (PICK)
    for (int t = tid >> 6; t < n.T; t += 16)
      pick_experts<NV>(z, how, n, t, l);
  __syncthreads();
  for (int a = tid; a < A; a += 1024)
    if (l.picked[a] >= 0) atomicAdd(&count[l.picked[a]], 1);
  __syncthreads();
  if (tid < 64) {  // first slot and first tile of every expert: a scan over the wave
    const int per = (n.experts + 63) / 64, e0 = tid * per, e1 = min(e0 + per, n.experts);
    int slots = 0, tiles = 0;
    for (int e = e0; e < e1; ++e) slots += (count[e] + 15) & ~15, tiles += (count[e] + rows - 1) / rows;
    const int own_s = slots, own_t = tiles;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int a = __shfl_up(slots, o), b = __shfl_up(tiles, o);
      if (tid >= o) slots += a, tiles += b;
    }
    if (tid == 63) total = tiles;
    slots -= own_s, tiles += st - own_t;
    for (int e = e0; e < e1; ++e) {
      next[e] = slots;
      for (int r = 0; r < count[e]; r += rows)
        l.tiles[tiles++] = MoeTile{e, slots + r, min(rows, count[e] - r), 0};
      slots += (count[e] + 15) & ~15;
    }
  }
  __syncthreads();
  for (int i = tid; i < st; i += 1024)
    l.tiles[i] = MoeTile{n.experts, i * rows, min(rows, n.T - i * rows), 0};
  if (tid == 0) *l.num_tiles = st + total;
  for (int a = tid; a < A; a += 1024) {
    if (l.picked[a] < 0) {
      l.at[a] = -1;
      continue;
    }
    const int slot = atomicAdd(&next[l.picked[a]], 1);
    l.slot_token[slot] = a / n.top;
    l.at[a] = slot;
  }
}

template <class How>
static hipError_t route(const Partials &z, How how, const MoeSizes &n, const MoeLists &l, hipStream_t s) {
  if (n.T <= 0) return hipSuccess;
  const int cols = n.experts + n.identity;
  if (n.experts < 1 || n.identity < 0 || cols > kMoeMaxExperts || n.top < 1 ||
      n.top > std::min(cols, kMoeMaxTop) || z.S < 1 || z.S > 8 || z.NP < cols ||
      (n.shared && n.gate_col >= z.NP) || (n.identity && !l.own))
    return hipErrorInvalidValue;
  const int rows = n.tile_rows();
#define FFMI_MR(NV)                                                                                          \
  do {                                                                                                       \
    if (n.T <= 64) {                                                                                         \
      hipLaunchKernelGGL((moe_lists_kernel<NV, true, How>), dim3(1), dim3(1024), 0, s, z, how, n, l, rows);  \
    } else {                                                                                                 \
      hipLaunchKernelGGL((moe_pick_kernel<NV, How>), dim3((n.T + 3) / 4), dim3(256), 0, s, z, how, n, l);    \
      hipLaunchKernelGGL((moe_lists_kernel<1, false, How>), dim3(1), dim3(1024), 0, s, z, how, n, l, rows);  \
    }                                                                                                        \
  } while (0)
  if (cols <= 64) FFMI_MR(1);
  else if (cols <= 128) FFMI_MR(2);
  else if (cols <= 256) FFMI_MR(4);
  else FFMI_MR(16);
#undef FFMI_MR
  return hipGetLastError();
}
hipError_t launch_moe_route(const Partials &z, const float *bias, const MoeSizes &n, const MoeLists &l,
                            hipStream_t s) {
  if (n.identity) return hipErrorInvalidValue;
  return route(z, bias, n, l, s);
}
hipError_t launch_moe_route_scores(const Partials &z, const MoeScores &sc, const MoeSizes &n, const MoeLists &l,
                                   hipStream_t s) {
  const int cols = n.experts + n.identity;
  if (sc.groups < 1 || cols % sc.groups || sc.keep < 1 || sc.keep > sc.groups ||
      n.top > cols / sc.groups * sc.keep || n.shared || !sc.correction)
    return hipErrorInvalidValue;
  return route(z, sc, n, l, s);
}

// ---------------------------------------------------------------------------
// products by expert
// ---------------------------------------------------------------------------
__device__ __forceinline__ f4 moe_mma(h8 a, h8 b, f4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf8, a), __builtin_bit_cast(bf8, b), c, 0,
                                                 0, 0);
}
__device__ __forceinline__ void store_bf16x4(uint16_t *p, float a, float b, float c, float d) {
  *reinterpret_cast<uint2 *>(p) =
      make_uint2(f2bf(a) | ((uint32_t)f2bf(b) << 16), f2bf(c) | ((uint32_t)f2bf(d) << 16));
}
// four consecutive output columns n.. of slot row m; gated: of the gate and up sums
// (f: the row's factor)
__device__ __forceinline__ float moe_unit(float gate, float up, float limit) {
  return limit > 0.f ? clamped_glu(gate, up, limit) : silu_glu(gate, up);
}
template <bool GATED>
__device__ __forceinline__ void moe_store(const MoeGroup &g, int m, int n, float f, float limit, const f4 &a,
                                          const f4 &b) {
  uint16_t *Y = (uint16_t *)g.Y;
  if constexpr (GATED)
    store_bf16x4(Y + act_packed_off(m, n, g.ldy), f * moe_unit(a[0], b[0], limit), f * moe_unit(a[1], b[1], limit),
                 f * moe_unit(a[2], b[2], limit), f * moe_unit(a[3], b[3], limit));
  else
    store_bf16x4(Y + (size_t)m * g.N + n, a[0], a[1], a[2], a[3]);
}

// Up to 16 rows: a workgroup has two 16-column tiles (a gate / up pair) and splits
// K over its four waves; weights straight to registers, U k-steps in flight.
template <bool GATED, bool NTL>
__global__ __launch_bounds__(256) void moe_few_kernel(MoeGemm a, int first, size_t wts) {
  constexpr int U = 8;
  __shared__ f4 red[3][2][64];
  if (first + (int)blockIdx.y >= *a.num_tiles) return;
  const MoeTile tl = a.tiles[first + blockIdx.y];
  const bool shared = tl.expert >= a.experts;
  const MoeGroup &g = a.g[shared];
  const int KT = g.K >> 5, ntiles = (GATED ? 2 : 1) * (g.N >> 4), tile0 = blockIdx.x * 2;
  if (tile0 >= ntiles) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, m = lane & 15;
  const size_t wks = wts == 512 ? (size_t)ntiles * 512 : 512, ts = wts == 512 ? 512 : (size_t)KT * 512;
  const uint16_t *W = (const uint16_t *)g.W + (shared ? 0 : tl.expert * g.w_stride) + lane * 8;
  const uint16_t *w0 = W + tile0 * ts, *w1 = W + min(tile0 + 1, ntiles - 1) * ts;
  const uint16_t *x;
  if constexpr (GATED) {
    const int slot = tl.slot0 + min(m, tl.rows - 1);
    x = (const uint16_t *)g.X + (size_t)(shared ? slot : a.slot_token[slot]) * g.K + 8 * (lane >> 4);
  } else {
    x = (const uint16_t *)g.X + ((size_t)(tl.slot0 >> 4) * KT * 64 + lane) * 8;
  }
  constexpr int XS = GATED ? 32 : 512;
  const int per = (KT + 3) / 4, kb = min(KT, wave * per), ke = min(KT, kb + per);
  f4 acc[2];
  acc[0] = acc[1] = f4{0.f, 0.f, 0.f, 0.f};
  const h8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  for (int k = kb; k < ke; k += U) {
    h8 b[U][2], xv[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const size_t kk = min(k + u, ke - 1);
      b[u][0] = ld_weight<NTL>(w0 + kk * wks), b[u][1] = ld_weight<NTL>(w1 + kk * wks);
      xv[u] = *reinterpret_cast<const h8 *>(x + kk * XS);
    }
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (k + u >= ke) xv[u] = zero;
      acc[0] = moe_mma(b[u][0], xv[u], acc[0]);  // D = W . X^T: a lane has 4 columns of a row
      acc[1] = moe_mma(b[u][1], xv[u], acc[1]);
    }
  }
  if (wave > 0) red[wave - 1][0][lane] = acc[0], red[wave - 1][1][lane] = acc[1];
  __syncthreads();
  if (wave > 0) return;
#pragma unroll
  for (int w = 0; w < 3; ++w) acc[0] += red[w][0][lane], acc[1] += red[w][1][lane];
  if (m >= tl.rows) return;
  const int row = tl.slot0 + m, n = (lane >> 4) * 4;
  if constexpr (GATED) {
    moe_store<true>(g, row, blockIdx.x * 16 + n, shared ? a.gate[row] : 1.0f, a.limit, acc[0], acc[1]);
  } else {
    moe_store<false>(g, row, tile0 * 16 + n, 1.0f, 0.f, acc[0], acc[0]);
    if (tile0 + 1 < ntiles) moe_store<false>(g, row, tile0 * 16 + 16 + n, 1.0f, 0.f, acc[1], acc[1]);
  }
}

// Up to 256 rows x 16 tiles a workgroup: eight waves as 2 (every other 16 rows) x 4
// (weight tiles); both operands' fragments go to LDS as they are stored (row-major
// rows: a lane fetches its own row's 16 bytes), NB - 1 k-steps in flight across raw
// barriers with counted waits, as the dense tile product does.  NF: 16-row fragments
// of a wave that hold rows; with up to 128 rows the other half is not fetched either.
template <bool GATED, int NF, int NB>
__device__ __forceinline__ void moe_tile(const MoeGemm &a, const MoeTile &tl, int tile0, size_t wts,
                                         h8 (*lds)[32][64]) {
  constexpr int OPS = NF > 4 ? 4 : 3;  // fragments that a wave fetches for a k-step
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const bool shared = tl.expert >= a.experts;
  const MoeGroup &g = a.g[shared];
  const int KT = g.K >> 5, ntiles = (GATED ? 2 : 1) * (g.N >> 4);
  const size_t wks = wts == 512 ? (size_t)ntiles * 512 : 512, ts = wts == 512 ? 512 : (size_t)KT * 512;
  const uint16_t *W = (const uint16_t *)g.W + (shared ? 0 : tl.expert * g.w_stride) + lane * 8;
  const uint16_t *src[OPS];
#pragma unroll
  for (int p = 0; p < OPS; ++p) {
    const int f = wave + 8 * p;
    if (p >= OPS - 2) {  // weight tiles
      src[p] = W + min(tile0 + f - 8 * (OPS - 2), ntiles - 1) * ts;
    } else if (GATED) {
      const int slot = tl.slot0 + min(f * 16 + (lane & 15), tl.rows - 1);
      src[p] = (const uint16_t *)g.X + (size_t)(shared ? slot : a.slot_token[slot]) * g.K + 8 * (lane >> 4);
    } else {
      const int mt = (tl.slot0 >> 4) + min(f, (tl.rows - 1) >> 4);
      src[p] = (const uint16_t *)g.X + ((size_t)mt * KT * 64 + lane) * 8;
    }
  }
  auto issue_one = [&](int kt, int p) {
    const bool w = p >= OPS - 2;
    __builtin_amdgcn_global_load_lds(
        (const __attribute__((address_space(1))) void *)(src[p] + (size_t)kt * (w ? wks : GATED ? 32 : 512)),
        (__attribute__((address_space(3))) void *)(&lds[kt % NB][wave + 8 * (w ? p - (OPS - 2) + 2 : p)][0]), 16,
        0, 0);
  };
  const int wm = wave >> 2, wn = wave & 3;
  f4 acc[NF][4];
#pragma unroll
  for (int i = 0; i < NF; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int kt = 0; kt < NB - 1; ++kt)
    if (kt < KT)
#pragma unroll
      for (int p = 0; p < OPS; ++p) issue_one(kt, p);
  static_assert(NB == 4, "the waits below count NB - 2 younger stages");
  for (int kt = 0; kt < KT; ++kt) {
    // step kt has arrived once at most the younger steps' loads remain; the barrier
    // makes every wave's visible and retires the reads of the buffer filled next
    const int ahead = min(KT - 1 - kt, NB - 2);
    if (ahead >= 2) {
      if constexpr (OPS == 4) asm volatile("s_waitcnt vmcnt(8)" ::: "memory");
      else asm volatile("s_waitcnt vmcnt(6)" ::: "memory");
    } else if (ahead == 1) {
      if constexpr (OPS == 4) asm volatile("s_waitcnt vmcnt(4)" ::: "memory");
      else asm volatile("s_waitcnt vmcnt(3)" ::: "memory");
    } else {
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    const bool more = kt + NB - 1 < KT;
    const int buf = kt % NB;
    h8 xf[NF], wf[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) wf[j] = lds[buf][16 + wn * 4 + j][lane];
#pragma unroll
    for (int i = 0; i < NF; ++i) xf[i] = lds[buf][2 * i + wm][lane];
#pragma unroll
    for (int i = 0; i < NF; ++i) {
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[i][j] = moe_mma(wf[j], xf[i], acc[i][j]);
      if (more)
#pragma unroll
        for (int p = 0; p < OPS; ++p)  // (spread: a fetch's issue hides under the products)
          if (p * NF / OPS == i) issue_one(kt + NB - 1, p);
    }
  }
#pragma unroll
  for (int i = 0; i < NF; ++i) {
    const int m = (2 * i + wm) * 16 + (lane & 15);
    if (m >= tl.rows) continue;
    const float f = GATED && shared ? a.gate[tl.slot0 + m] : 1.0f;
#pragma unroll
    for (int j = 0; j < 4; j += GATED ? 2 : 1) {
      const int tile = tile0 + wn * 4 + j;
      if (tile >= ntiles) continue;
      moe_store<GATED>(g, tl.slot0 + m, (GATED ? tile >> 1 : tile) * 16 + (lane >> 4) * 4, f, a.limit,
                       acc[i][j], acc[i][GATED ? j + 1 : j]);
    }
  }
}
// The shared expert's workgroups first (the longest), their row tiles of a column
// tile on one XCD; then the experts', a row tile's columns in turn.
template <bool GATED>
__global__ __launch_bounds__(512, 1) void moe_tile_kernel(MoeGemm a, int first, int st, int cols_shared,
                                                          int cols, size_t wts) {
  __shared__ __attribute__((aligned(1024))) h8 lds[4][32][64];
  const int nsh = st * cols_shared, b = blockIdx.x;
  int tile, col;
  if (b < nsh) {
    const int xcd = b & 7, q = nsh >> 3, r = nsh & 7;
    const int L = (xcd < r ? xcd * (q + 1) : r * (q + 1) + (xcd - r) * q) + (b >> 3);
    tile = L % st, col = L / st;
  } else {
    tile = first + st + (b - nsh) / cols, col = (b - nsh) % cols;
    if (tile >= *a.num_tiles) return;
  }
  const MoeTile tl = a.tiles[tile];
  const int frags = (tl.rows + 15) >> 4;
  if (frags <= 4) moe_tile<GATED, 2, 4>(a, tl, col * 16, wts, lds);
  else if (frags <= 8) moe_tile<GATED, 4, 4>(a, tl, col * 16, wts, lds);
  else if (frags <= 12) moe_tile<GATED, 6, 4>(a, tl, col * 16, wts, lds);
  else moe_tile<GATED, 8, 4>(a, tl, col * 16, wts, lds);
}

// fp32: 16 rows x 64 columns a workgroup
template <bool GATED>
__global__ __launch_bounds__(256) void moe_f32_kernel(MoeGemm a, int first) {
  __shared__ float sx[16][33], sw[GATED ? 2 : 1][64][33];
  if (first + (int)blockIdx.y >= *a.num_tiles) return;
  const MoeTile tl = a.tiles[first + blockIdx.y];
  const bool shared = tl.expert >= a.experts;
  const MoeGroup &g = a.g[shared];
  const int n0 = blockIdx.x * 64, tid = threadIdx.x, r = tid & 15, c = tid >> 4;
  if (n0 >= g.N) return;
  const float *W = (const float *)g.W + (shared ? 0 : tl.expert * g.w_stride);
  for (int m0 = 0; m0 < tl.rows; m0 += 16) {
    float acc[GATED ? 2 : 1][4];
#pragma unroll
    for (int p = 0; p < (GATED ? 2 : 1); ++p)
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[p][j] = 0.f;
    for (int k0 = 0; k0 < g.K; k0 += 32) {
      __syncthreads();
      for (int i = tid; i < 16 * 32; i += 256) {
        const int slot = tl.slot0 + min(m0 + i / 32, tl.rows - 1);
        sx[i / 32][i % 32] =
            ((const float *)g.X)[(size_t)(GATED && !shared ? a.slot_token[slot] : slot) * g.K + k0 + i % 32];
      }
#pragma unroll
      for (int p = 0; p < (GATED ? 2 : 1); ++p)
        for (int i = tid; i < 64 * 32; i += 256)
          sw[p][i / 32][i % 32] = W[((size_t)p * g.N + min(n0 + i / 32, g.N - 1)) * g.K + k0 + i % 32];
      __syncthreads();
#pragma unroll
      for (int k = 0; k < 32; ++k)
#pragma unroll
        for (int p = 0; p < (GATED ? 2 : 1); ++p)
#pragma unroll
          for (int j = 0; j < 4; ++j) acc[p][j] = fmaf(sx[r][k], sw[p][c + 16 * j][k], acc[p][j]);
    }
    if (m0 + r < tl.rows)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int n = n0 + c + 16 * j;
        const int row = tl.slot0 + m0 + r;
        if (n >= g.N) continue;
        if constexpr (GATED)
          ((float *)g.Y)[(size_t)row * g.ldy + n] =
              (shared ? a.gate[row] : 1.0f) * moe_unit(acc[0][j], acc[GATED ? 1 : 0][j], a.limit);
        else
          ((float *)g.Y)[(size_t)row * g.N + n] = acc[0][j];
      }
  }
}

hipError_t launch_moe_gemm(const MoeGemm &a, const MoeSizes &n, bool gated, bool f32, bool stream_weights,
                           hipStream_t s) {
  if (n.T <= 0) return hipSuccess;
  const bool shared = gated && n.shared;
  int N = 0;
  for (int i = 0; i < (shared ? 2 : 1); ++i) {
    const MoeGroup &g = a.g[i];
    if (g.N % 32 || g.K % 32 || g.N <= 0 || g.K <= 0 || (gated && (g.ldy < g.N || g.ldy % 32)))
      return hipErrorInvalidValue;
    N = std::max(N, g.N);
  }
  // (the second product leaves the shared expert's tiles out)
  const int rows = n.tile_rows(), st = shared ? n.shared_tiles(rows) : 0, first = n.shared_tiles(rows) - st;
  const int tiles = n.expert_tiles(rows);
  if (st + tiles > 65535 || (shared && !a.gate)) return hipErrorInvalidValue;
  if (f32) {
    const dim3 grid((N + 63) / 64, st + tiles);
    if (gated) hipLaunchKernelGGL(moe_f32_kernel<true>, grid, dim3(256), 0, s, a, first);
    else hipLaunchKernelGGL(moe_f32_kernel<false>, grid, dim3(256), 0, s, a, first);
    return hipGetLastError();
  }
  const int per = gated ? 2 : 1;
  const size_t wts = weights_kmajor() ? 512 : 0;
  if (rows == kMoeMany) {
    const int cols = (per * a.g[0].N / 16 + 15) / 16, cols_shared = st ? (per * a.g[1].N / 16 + 15) / 16 : 0;
    const dim3 grid(st * cols_shared + tiles * cols);
    if (gated)
      hipLaunchKernelGGL(moe_tile_kernel<true>, grid, dim3(512), 0, s, a, first, st, cols_shared, cols, wts);
    else
      hipLaunchKernelGGL(moe_tile_kernel<false>, grid, dim3(512), 0, s, a, first, st, cols_shared, cols, wts);
    return hipGetLastError();
  }
  const dim3 grid((per * N / 16 + 1) / 2, st + tiles);
#define FFMI_MF(G, NL) hipLaunchKernelGGL((moe_few_kernel<G, NL>), grid, dim3(256), 0, s, a, first, wts)
  if (gated && stream_weights) FFMI_MF(true, true);
  else if (gated) FFMI_MF(true, false);
  else if (stream_weights) FFMI_MF(false, true);
  else FFMI_MF(false, false);
#undef FFMI_MF
  return hipGetLastError();
}

}  // namespace ffmi
