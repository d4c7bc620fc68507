// memory.hip -- matrix memories, token by token (memory.h).
#include "memory_util.h"

#include <algorithm>
#include <type_traits>

namespace ffmi {

namespace {

constexpr int NT = 512, NW = NT / 64;

// 8 elements of a row in registers, and their product with 8 fp32 values
struct Row8 {
  uint4 v;
  __device__ __forceinline__ void load(const uint16_t *p) { v = *reinterpret_cast<const uint4 *>(p); }
  __device__ __forceinline__ float dot(const float *x) const {
    f4 a, b;
    unpack8_bf16(v, a, b);
    const f4 u = *reinterpret_cast<const f4 *>(x), w = *reinterpret_cast<const f4 *>(x + 4);
    return fmaf(a[0], u[0], fmaf(a[1], u[1], fmaf(a[2], u[2], a[3] * u[3]))) +
           fmaf(b[0], w[0], fmaf(b[1], w[1], fmaf(b[2], w[2], b[3] * w[3])));
  }
};
struct Row8F {
  f4 a, b;
  __device__ __forceinline__ void load(const float *p) {
    a = *reinterpret_cast<const f4 *>(p), b = *reinterpret_cast<const f4 *>(p + 4);
  }
  __device__ __forceinline__ float dot(const float *x) const {
    const f4 u = *reinterpret_cast<const f4 *>(x), w = *reinterpret_cast<const f4 *>(x + 4);
    return fmaf(a[0], u[0], fmaf(a[1], u[1], fmaf(a[2], u[2], a[3] * u[3]))) +
           fmaf(b[0], w[0], fmaf(b[1], w[1], fmaf(b[2], w[2], b[3] * w[3])));
  }
};
// A narrow second product: four lanes a row, 32 columns at a time.  The first rows' first
// 32 kAhead columns are fetched ahead (head), before the product's input is there.
template <class E, int kAhead>
struct LowRankRows {
  typedef typename std::conditional<sizeof(E) == 2, Row8, Row8F>::type Row;
  static constexpr int kRows = NT / 4;
  Row head[kAhead ? kAhead : 1];
  static __device__ __forceinline__ const E *row(const LowRank &l, int r) {
    return (const E *)l.w + (size_t)r * l.r + (threadIdx.x & 3) * 8;
  }
  __device__ __forceinline__ void fetch(const LowRank &l, int row0, int n) {
    const int c = min((int)threadIdx.x >> 2, n - 1);
#pragma unroll
    for (int i = 0; i < kAhead; ++i)
      if (i * 32 < l.r) head[i].load(row(l, row0 + c) + i * 32);
  }
  // rows [row0, row0 + n) for np tokens whose inputs are in LDS (x [np][r])
  template <class D>
  __device__ __forceinline__ void run(const LowRank &l, int row0, int n, int np, const float *x, D done) {
    const int j = threadIdx.x & 3;
    for (int c0 = 0; c0 < n; c0 += kRows) {
      const int c = c0 + ((int)threadIdx.x >> 2), cc = min(c, n - 1);
      const E *w = row(l, row0 + cc);
      Row cur[kAhead ? kAhead : 1];
#pragma unroll
      for (int i = 0; i < kAhead; ++i) {
        cur[i] = head[i];
        if (c0 > 0 && i * 32 < l.r) cur[i].load(w + i * 32);
      }
#pragma unroll 1
      for (int t = 0; t < np; ++t) {
        const float *xt = x + t * l.r + j * 8;
        float v = 0.f;
#pragma unroll
        for (int i = 0; i < kAhead; ++i)
          if (i * 32 < l.r) v += cur[i].dot(xt + i * 32);
#pragma unroll 1
        for (int k = kAhead * 32; k < l.r; k += 32) {
          Row more;
          more.load(w + k);
          v += more.dot(xt + k);
        }
        v += __shfl_xor(v, 1);
        v += __shfl_xor(v, 2);
        if (j == 0 && c < n) done(t, c, v);
      }
    }
  }
};

// LDS of a piece of tokens, in floats
__host__ __device__ inline int piece_floats(const Memory &a) {
  return 3 * a.dg + 2 * a.vs + a.vg + a.decay.r + a.gate.r + 8;
}

// A workgroup per (head, span, part of the state's columns: `cols` of them).  The columns
// in slices of 4 << cw, a slice in registers: thread = (4 columns, every (NT >> cw)-th
// row), P rows a thread; tokens in pieces that fit the LDS.  Per piece: projections,
// convolution, gates and norms of all its tokens; then slice by slice the tokens in turn,
// one barrier each (two sets of partial sums alternate); then the outputs' norm and gate.
// SPLIT: more than one part; outputs (and m) are left in scratch instead.
// What memory has to give comes in the order it is waited for: narrow matrices, the
// products' columns, the state.
template <MemoryRule RULE, class E, int P, bool SPLIT>
__global__ __launch_bounds__(NT, SPLIT ? 4 : 2) void memory_steps_kernel(const char *__restrict__ blob, int off_spans, Memory a,
                                                          MemoryScratch w, int limit, int piece, int cw, int cols) {
  constexpr bool CONV = RULE == kMemoryDelta;
  constexpr int TAPS = CONV ? 4 : 1;  // up to here without a loop
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const PagedSpan sp = reinterpret_cast<const PagedSpan *>(blob + off_spans)[blockIdx.y];
  if (sp.n > limit) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.x;
  const int dg = a.dg, vs = a.vs, vg = a.vg, hq = h / (a.H / a.G), bank = sp.bank;
  const int cb = SPLIT ? blockIdx.z * cols : 0, ce = SPLIT ? min(cb + cols, vs) : vs;
  const int CW = 1 << cw, SW = CW * 4, NG = NT >> cw;
  const int r1 = a.decay.r, r2 = SPLIT ? 0 : a.gate.r;
  float *sq = lds, *sk = sq + piece * dg, *sg = sk + piece * dg, *sv = sg + piece * dg, *so = sv + piece * vs;
  float *sgate = so + piece * vs, *sx = sgate + piece * vg, *sx2 = sx + piece * r1;
  float *scal = sx2 + piece * a.gate.r;  // [token][8]: beta or i, f, k . q, m
  float *red = scal + piece * 8;         // [2][2][NW][SW]
  const int cl = (tid & (CW - 1)) * 4, rg = tid >> cw;
  const bool one = ce - cb <= SW;  // all the columns stay in registers
  const bool first = h % (a.H / a.G) == 0 && cb == 0;  // (query and key heads are shared)
  float *S = a.state + ((size_t)sp.slot * a.H + h) * dg * vs;

  LowRankRows<E, SPLIT ? 0 : 4> decay, gate;
  if constexpr (RULE != kMemoryNormed) decay.fetch(a.decay, h * a.dim, a.dim);
  if (r2 > 0) gate.fetch(a.gate, h * a.vdim, a.vdim);
  const float rate = RULE == kMemoryDelta ? a.rate[h] : 0.f;
  float dbias = 0.f;  // of the first row that this thread finishes
  if constexpr (RULE != kMemoryNormed) dbias = a.dbias[(size_t)h * dg + min(tid >> 2, a.dim - 1)];
  float nw[4];  // the norm's weights of this lane's columns
  if constexpr (!SPLIT)
#pragma unroll
    for (int i = 0; i < 4; ++i) nw[i] = a.norm[(a.norm_heads ? h * vg : 0) + min(lane + 64 * i, vg - 1)];
  float m = 0.f;
  if constexpr (RULE == kMemoryNormed)
    if (sp.pos0 > 0) m = a.peak[((size_t)sp.slot * 2 + bank) * a.H + h];

  f4 st[P];
  auto load = [&](int c0, bool fresh) {
#pragma unroll
    for (int p = 0; p < P; ++p) {
      const int row = p * NG + rg;
      st[p] = f4{0.f, 0.f, 0.f, 0.f};
      if (!fresh && row < dg && c0 + cl < ce) st[p] = *reinterpret_cast<const f4 *>(S + (uint32_t)(row * vs + c0 + cl));
    }
  };
  auto store = [&](int c0) {
#pragma unroll
    for (int p = 0; p < P; ++p) {
      const int row = p * NG + rg;
      if (row < dg && c0 + cl < ce) *reinterpret_cast<f4 *>(S + (uint32_t)(row * vs + c0 + cl)) = st[p];
    }
  };

  const size_t slab = (size_t)a.T * a.y.NP, C = memory_columns(a);
  const int past = max(a.taps - 1, 0);
  const float *old = a.carry + ((size_t)sp.slot * 2 + bank) * past * C;
  float *now = a.carry + ((size_t)sp.slot * 2 + (bank ^ 1)) * past * C;
  // A column of the first product for one token, with what its convolution reads: asked for
  // (fetch), then finished.
  struct Item {
    int t, c, y;  // token of the piece, item, column (-1: none)
    float u, x[CONV ? TAPS - 1 : 1], w[TAPS];
  };
  // the row d tokens before token t, column c of q | k | v
  auto before = [&](int t, int d, int c) {
    if (t < d) return old[(d - t - 1) * C + c];
    return sum_at(a.y, slab, (size_t)(sp.t0 + t - d) * a.y.NP + a.col + c);
  };
  // what a token needs of the first product, item by item: its column, and where it goes
  const int nv = ce - cb, e1 = 2 * dg, e2 = e1 + nv, e3 = e2 + r1 + r2, e4 = e3 + (SPLIT || r2 > 0 ? 0 : vg);
  const int items = e4 + (RULE == kMemoryDelta ? 1 : RULE == kMemoryNormed ? 2 : 0);
  auto column = [&](int c) {
    if (c < e1) return a.col + (c < dg ? hq * dg + c : (a.G + hq) * dg + c - dg);
    if (c < e2) return cb + c - e1 < vg ? a.col + 2 * a.G * dg + h * vg + cb + c - e1 : -1;
    if (c < e3) return c - e2 < r1 ? a.decay.col + c - e2 : a.gate.col + c - e2 - r1;
    if (c < e4) return a.col_gate + h * vg + c - e3;
    return RULE == kMemoryDelta ? a.col_beta + h : (c == e4 ? a.col_i : a.col_f) + h;
  };
  auto fetch = [&](int p0, int np, int id) {
    Item it;
    it.t = id / items, it.c = id - it.t * items, it.y = id < np * items ? column(it.c) : -1, it.u = 0.f;
    const int t = p0 + it.t, n = min(past, sp.pos0 + t), c = it.y - a.col;
    if (it.y >= 0) it.u = sum_at(a.y, slab, (size_t)(sp.t0 + t) * a.y.NP + it.y);
    const bool conv = past < TAPS && it.c < e2 && it.y >= 0;
    if constexpr (CONV)
#pragma unroll
      for (int d = 0; d < TAPS; ++d) {
        it.w[d] = 0.f;
        if (d > 0) it.x[d - 1] = 0.f;
        if (conv && d < a.taps) it.w[d] = a.conv[(past - d) * C + c];
        if (d > 0 && conv && d <= n) it.x[d - 1] = before(t, d, c);
      }
    return it;
  };
  // through the convolution and the activation; keep: this workgroup carries the row on
  auto project = [&](const Item &it, int t, bool keep) {
    if (it.y < 0) return 0.f;
    float v = it.u;
    if (CONV && a.taps > 0) {
      const int c = it.y - a.col;
      if (past < TAPS) {
        v *= it.w[0];
#pragma unroll
        for (int d = 1; d < TAPS; ++d) v = fmaf(it.x[d - 1], it.w[d], v);
        if (keep && t == 0)  // (a short span: earlier rows move on)
#pragma unroll
          for (int d = 1; d < TAPS; ++d)
            if (sp.n + d - 1 < past) now[(sp.n + d - 1) * C + c] = it.x[d - 1];
      } else {
        v *= a.conv[past * C + c];
        for (int d = 1; d <= min(past, sp.pos0 + t); ++d) v = fmaf(before(t, d, c), a.conv[(past - d) * C + c], v);
        if (keep && t == 0)
          for (int p = sp.n; p < past; ++p) now[p * C + c] = p - sp.n < sp.pos0 ? old[(p - sp.n) * C + c] : 0.f;
      }
      if (keep && sp.n - 1 - t < past) now[(sp.n - 1 - t) * C + c] = it.u;
    }
    return a.silu ? silu_f(v) : v;
  };
  auto finish = [&](int p0, const Item &it) {
    const int t = it.t, c = it.c;
    const float u = it.u;
    if (c < e1) {
      (c < dg ? sq : sk)[t * dg + (c < dg ? c : c - dg)] = project(it, p0 + t, first);
    } else if (c < e2) {
      const int vc = cb + c - e1;
      sv[t * vs + vc] = RULE == kMemoryNormed && vc == a.vdim ? 1.f : project(it, p0 + t, true);
    } else if (c < e3) {
      if (c - e2 < r1) sx[t * r1 + c - e2] = u;
      else sx2[t * r2 + c - e2 - r1] = u;
    } else if (c < e4) {
      sgate[t * vg + c - e3] = u;
    } else if constexpr (RULE == kMemoryDelta) {
      scal[t * 8] = sigmoid_f(u);
    } else if constexpr (RULE == kMemoryNormed) {
      const float z = a.cap * tanhf(__fdiv_rn(u + (c == e4 ? a.bi : a.bf)[h], a.cap));
      scal[t * 8 + c - e4] = c == e4 ? z : -softplus_f(-z);
    }
  };
  int turn = 0;
  for (int p0 = 0; p0 < sp.n; p0 += piece) {
    const int np = min(piece, sp.n - p0);
    if constexpr (SPLIT) {
      for (int id = tid; id < np * items; id += NT) {
        const Item it = fetch(p0, np, id);
        if (p0 == 0 && id == tid) load(cb, sp.pos0 == 0);
        finish(p0, it);
      }
    } else {
      for (int id = tid; id < np * items; id += 2 * NT) {  // two at a time
        const Item i0 = fetch(p0, np, id), i1 = fetch(p0, np, id + NT);
        if (p0 == 0 && id == tid) load(cb, sp.pos0 == 0);
        finish(p0, i0);
        if (id + NT < np * items) finish(p0, i1);
      }
    }
    if (p0 == 0 && tid >= np * items) load(cb, sp.pos0 == 0);
    __syncthreads();
    // gates, norms
    if constexpr (RULE == kMemoryNormed) {
      float mm = m;  // (every wave follows m for its own tokens)
      for (int t = 0; t < np; ++t) {
        const float i = scal[t * 8], f = scal[t * 8 + 1], mn = fmaxf(f + mm, i);
        if (t % NW == wave) {
          const float d = expf(f + mm - mn), kf = expf(i - mn);
          if (lane == 0) scal[t * 8 + 3] = mn;
          for (int c = lane; c < dg; c += 64) {
            sg[t * dg + c] = d;
            sq[t * dg + c] *= a.q_scale;
            sk[t * dg + c] *= kf;
          }
        }
        mm = mn;
      }
      m = mm;
    } else {
      for (int t = wave; t < np; t += NW) {
        float fq = a.q_scale, fk = 1.f;
        if (a.unit || RULE == kMemoryDelta) {
          float qq = 0.f, kk = 0.f, kq = 0.f;
          for (int c = lane; c < dg; c += 64) {
            const float x = sq[t * dg + c], y = sk[t * dg + c];
            qq = fmaf(x, x, qq), kk = fmaf(y, y, kk), kq = fmaf(x, y, kq);
          }
#pragma unroll
          for (int o = 32; o > 0; o >>= 1)
            qq += __shfl_xor(qq, o), kk += __shfl_xor(kk, o), kq += __shfl_xor(kq, o);
          if (a.unit)
            fq *= __fdiv_rn(1.0f, sqrtf(qq + 1e-6f)), fk = __fdiv_rn(1.0f, sqrtf(kk + 1e-6f));
          if (lane == 0) scal[t * 8 + 2] = kq * fq * fk;
        }
        for (int c = lane; c < dg; c += 64) {
          sq[t * dg + c] *= fq;
          sk[t * dg + c] *= fk;
        }
      }
      decay.run(a.decay, h * a.dim, a.dim, np, sx,
                [&](int t, int c, float z) {
                  z += c == tid >> 2 ? dbias : a.dbias[(size_t)h * dg + c];
                  sg[t * dg + c] = sizeof(E) == 2 ? ex2(log2_decay<RULE>(a, rate, z)) : decay_of<RULE>(a, rate, z);
                });
      for (int id = tid; id < np * (dg - a.dim); id += NT)
        sg[id / (dg - a.dim) * dg + a.dim + id % (dg - a.dim)] = 1.f;
    }
    if (r2 > 0) gate.run(a.gate, h * a.vdim, a.vdim, np, sx2, [&](int t, int c, float z) { sgate[t * vg + c] = z; });
    __syncthreads();
    // the tokens in turn
    for (int c0 = cb; c0 < ce; c0 += SW) {
      if (!one && (p0 > 0 || c0 > cb)) load(c0, sp.pos0 + p0 == 0);
      const bool col = c0 + cl < ce;
      for (int t = 0; t < np; ++t, turn ^= 1) {
        float *part = red + turn * 2 * NW * SW;
        f4 v = f4{0.f, 0.f, 0.f, 0.f}, pk = v, pq = v;
        if (col) v = *reinterpret_cast<const f4 *>(sv + t * vs + c0 + cl);
#pragma unroll
        for (int p = 0; p < P; ++p) {
          const int row = p * NG + rg;
          if (row >= dg) continue;
          const float g = sg[t * dg + row], k = sk[t * dg + row], q = sq[t * dg + row];
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            if constexpr (RULE == kMemoryDelta) {
              st[p][e] *= g;
              pk[e] = fmaf(k, st[p][e], pk[e]);
            } else {
              st[p][e] = fmaf(g, st[p][e], k * v[e]);
            }
            pq[e] = fmaf(q, st[p][e], pq[e]);
          }
        }
        for (int o = CW; o < 64; o <<= 1)
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            pq[e] += __shfl_xor(pq[e], o);
            if constexpr (RULE == kMemoryDelta) pk[e] += __shfl_xor(pk[e], o);
          }
        if (lane < CW) {
          *reinterpret_cast<f4 *>(part + wave * SW + cl) = pq;
          if constexpr (RULE == kMemoryDelta) *reinterpret_cast<f4 *>(part + (NW + wave) * SW + cl) = pk;
        }
        __syncthreads();
        f4 u = v;
        if constexpr (RULE == kMemoryDelta) {
          f4 sum = *reinterpret_cast<const f4 *>(part + NW * SW + cl);
#pragma unroll
          for (int w = 1; w < NW; ++w) sum += *reinterpret_cast<const f4 *>(part + (NW + w) * SW + cl);
          u = (v - sum) * scal[t * 8];
#pragma unroll
          for (int p = 0; p < P; ++p) {
            const int row = p * NG + rg;
            if (row >= dg) continue;
            const float k = sk[t * dg + row];
#pragma unroll
            for (int e = 0; e < 4; ++e) st[p][e] = fmaf(k, u[e], st[p][e]);
          }
        }
        if (rg == 0 && col) {
          f4 o = *reinterpret_cast<const f4 *>(part + cl);
#pragma unroll
          for (int w = 1; w < NW; ++w) o += *reinterpret_cast<const f4 *>(part + w * SW + cl);
          if constexpr (RULE == kMemoryDelta) o += u * scal[t * 8 + 2];
          if constexpr (SPLIT)
            *reinterpret_cast<f4 *>(w.o + ((size_t)(sp.t0 + p0 + t) * a.H + h) * vs + c0 + cl) = o;
          else *reinterpret_cast<f4 *>(so + t * vs + c0 + cl) = o;
        }
      }
      if (!one || p0 + np >= sp.n) store(c0);
    }
    if constexpr (SPLIT) {
      if (RULE == kMemoryNormed && cb == 0 && tid < np)
        w.gates[((size_t)(sp.t0 + p0 + tid) * a.H + h) * 3 + 2] = scal[tid * 8 + 3];
    } else {
      __syncthreads();
      // a wave per token: norm and gate
      for (int t = wave; t < np; t += NW) {
        float f = 1.f, ss = 0.f;
        if constexpr (RULE == kMemoryNormed)
          f = __fdiv_rn(1.0f, fmaxf(fabsf(so[t * vs + a.vdim]), expf(-scal[t * 8 + 3])) + 1e-6f);
        for (int c = lane; c < a.vdim; c += 64) {
          const float v = so[t * vs + c] * f;
          ss = fmaf(v, v, ss);
        }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) ss += __shfl_xor(ss, o);
        const float r = f * inv_rms(ss, a.vdim, a.eps);
        const int row = sp.t0 + p0 + t;
        auto put = [&](int c, float wv) {
          const float gt = sgate[t * vg + c];
          const float v = c < a.vdim ? so[t * vs + c] * r * wv * (a.gate_silu ? silu_f(gt) : sigmoid_f(gt)) : 0.f;
          const int oc = a.out_col + h * vg + c;
          st_elem((E *)a.out + (sizeof(E) == 2 ? act_packed_off(row, oc, a.ldo) : (size_t)row * a.ldo + oc), v);
        };
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (lane + 64 * i < vg) put(lane + 64 * i, nw[i]);
        for (int c = lane + 256; c < vg; c += 64) put(c, a.norm[(a.norm_heads ? h * vg : 0) + c]);
      }
    }
    __syncthreads();
  }
  if constexpr (RULE == kMemoryNormed)
    if (tid == 0 && cb == 0) a.peak[((size_t)sp.slot * 2 + (bank ^ 1)) * a.H + h] = m;
}

bool bad_shape(const Memory &a) {
  return a.H < 1 || a.G < 1 || a.H % a.G || a.dg % 32 || a.vg % 32 || a.dg < a.dim || a.vg < a.vdim ||
         a.dim < 1 || a.vdim < 1 || a.vs != memory_state_columns(a.rule, a.vdim) || a.vs < a.vg ||
         a.dg > kMemoryMaxDim || a.vs > kMemoryMaxVdim + 32 || a.y.S < 1 || a.y.S > 8 || a.y.NP % 4 || a.col % 4 ||
         (a.rule == kMemoryDelta) != (a.taps > 0) || (a.taps > 0 && !a.conv) || (a.taps > 1 && !a.carry) || a.decay.r % 32 || a.gate.r % 32 ||
         (a.rule == kMemoryNormed ? !a.peak || !a.bi || !a.bf || a.decay.r : !a.decay.w || !a.dbias || !a.decay.r) ||
         (a.rule == kMemoryDelta && !a.rate) || !a.norm || !a.state || a.ldo % 32 || a.out_col % 32 ||
         a.out_col + a.H * a.vg > a.ldo;
}

template <MemoryRule RULE, class E>
hipError_t run_steps(const char *blob, int off_spans, int num_spans, const Memory &a, const MemoryScratch *w,
                     int limit, bool *left, hipStream_t s) {
  // the widest power of two of columns that leaves at most 8 rows a thread
  int cw = 3;
  while (cw < 6 && (4 << cw) < a.vs && ((a.dg << (cw + 1)) + NT - 1) / NT <= 8) ++cw;
  const int rows = ((a.dg << cw) + NT - 1) / NT;
  const int red = 2 * 2 * NW * (4 << cw), each = piece_floats(a), budget = 16 * 1024;  // floats of LDS
  const int piece = std::min({kShortSpan, limit, std::max(1, (budget - red) / each)});
  const size_t bytes = (size_t)(red + piece * each) * 4;
  if (bytes > 64 * 1024) return hipErrorInvalidValue;
  // few wide heads: their slices side by side
  const int slices = (a.vs + (4 << cw) - 1) / (4 << cw), wgs = a.H * num_spans;
  const int want = w && a.gate.r == 0 && sizeof(E) == 2 ? std::min(slices, (512 + wgs - 1) / wgs) : 1;
  const int cols = (slices + want - 1) / want * (4 << cw), parts = (a.vs + cols - 1) / cols;
  const MemoryScratch none;
  *left = parts > 1;
  const dim3 grid(a.H, num_spans, parts);
#define FFMI_MS(P)                                                                                                    \
  do {                                                                                                                \
    if constexpr (sizeof(E) == 2 && RULE != kMemoryDelta)                                                             \
      if (parts > 1) {                                                                                                \
        hipLaunchKernelGGL((memory_steps_kernel<RULE, E, P, true>), grid, dim3(NT), bytes, s, blob, off_spans, a, *w,  \
                           limit, piece, cw, cols);                                                                   \
        break;                                                                                                        \
      }                                                                                                               \
    hipLaunchKernelGGL((memory_steps_kernel<RULE, E, P, false>), grid, dim3(NT), bytes, s, blob, off_spans, a,        \
                       w ? *w : none, limit, piece, cw, cols);                                                        \
  } while (0)
  if (rows <= 1) FFMI_MS(1);
  else if (rows <= 2) FFMI_MS(2);
  else if (rows <= 4) FFMI_MS(4);
  else if (rows <= 8) FFMI_MS(8);
  else return hipErrorInvalidValue;
#undef FFMI_MS
  return hipGetLastError();
}

}  // namespace

hipError_t launch_memory_steps(const char *blob, int off_spans, int num_spans, const Memory &a,
                               const MemoryScratch *w, bool f32, int limit, bool *left, hipStream_t s) {
  *left = false;
  if (num_spans <= 0) return hipSuccess;
  if (bad_shape(a) || limit < 1 || (w && (!w->o || (a.rule == kMemoryNormed && !w->gates)))) return hipErrorInvalidValue;
#define FFMI_MR(RULE)                                                                              \
  return f32 ? run_steps<RULE, float>(blob, off_spans, num_spans, a, w, limit, left, s)            \
             : run_steps<RULE, uint16_t>(blob, off_spans, num_spans, a, w, limit, left, s)
  if (a.rule == kMemoryGated) FFMI_MR(kMemoryGated);
  if (a.rule == kMemoryDelta) FFMI_MR(kMemoryDelta);
  FFMI_MR(kMemoryNormed);
#undef FFMI_MR
}

}  // namespace ffmi
