// memory.hip -- matrix memories, token by token (memory.h).
#include "memory_util.h"

#include <algorithm>

namespace ffmi {

namespace {

constexpr int NT = 512, NW = NT / 64;

__device__ __forceinline__ float dot_part(const uint16_t *w, const float *x) {
  const uint2 v = *reinterpret_cast<const uint2 *>(w);
  const f4 u = *reinterpret_cast<const f4 *>(x);
  return fmaf(__builtin_bit_cast(float, v.x << 16), u[0],
              fmaf(__builtin_bit_cast(float, v.x & 0xffff0000u), u[1],
                   fmaf(__builtin_bit_cast(float, v.y << 16), u[2],
                        __builtin_bit_cast(float, v.y & 0xffff0000u) * u[3])));
}
__device__ __forceinline__ float dot_part(const float *w, const float *x) {
  const f4 v = *reinterpret_cast<const f4 *>(w), u = *reinterpret_cast<const f4 *>(x);
  return fmaf(v[0], u[0], fmaf(v[1], u[1], fmaf(v[2], u[2], v[3] * u[3])));
}
// rows [row0, row0 + n) of a second product, for np tokens whose inputs are in LDS
// (x [np][r]): done(token, row, value); eight lanes a row
template <class E, class D>
__device__ __forceinline__ void low_rank(const LowRank &l, int row0, int n, int np, const float *x, D done) {
  const int j = threadIdx.x & 7;
  for (int id = threadIdx.x >> 3; id < np * n; id += NT / 8) {
    const int t = id / n, c = id - t * n;
    const E *w = (const E *)l.w + (size_t)(row0 + c) * l.r + j * 4;
    float v = 0.f;
    for (int k = 0; k < l.r; k += 32) v += dot_part(w + k, x + t * l.r + j * 4 + k);
#pragma unroll
    for (int o = 1; o < 8; o <<= 1) v += __shfl_xor(v, o);
    if (j == 0) done(t, c, v);
  }
}

// LDS of a piece of tokens, in floats
__host__ __device__ inline int piece_floats(const Memory &a) {
  return 3 * a.dg + 2 * a.vs + a.vg + a.decay.r + a.gate.r + 8;
}

// A workgroup per (head, span).  The state's columns in slices of 4 << cw, a slice in
// registers: thread = (4 columns, every (NT >> cw)-th row), P rows a thread; tokens in
// pieces that fit the LDS.  Per piece: projections, convolution, gates and norms of all
// its tokens; then slice by slice the tokens in turn, one barrier each (two sets of
// partial sums alternate); then the outputs' norm and gate.
template <MemoryRule RULE, class E, int P>
__global__ __launch_bounds__(NT) void memory_steps_kernel(const char *__restrict__ blob, int off_spans, Memory a,
                                                          int limit, int piece, int cw) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const PagedSpan sp = reinterpret_cast<const PagedSpan *>(blob + off_spans)[blockIdx.y];
  if (sp.n > limit) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.x;
  const int dg = a.dg, vs = a.vs, vg = a.vg, hq = h / (a.H / a.G);
  const int CW = 1 << cw, SW = CW * 4, NG = NT >> cw;
  float *sq = lds, *sk = sq + piece * dg, *sg = sk + piece * dg, *sv = sg + piece * dg, *so = sv + piece * vs;
  float *sgate = so + piece * vs, *sx = sgate + piece * vg, *sx2 = sx + piece * a.decay.r;
  float *scal = sx2 + piece * a.gate.r;  // [token][8]: beta or i, f, k . q, m, key factor, decay
  float *red = scal + piece * 8;         // [2][2][NW][SW]
  const int cl = (tid & (CW - 1)) * 4, rg = tid >> cw;
  const bool one = vs <= SW;  // the whole state stays in registers
  float *S = a.state + ((size_t)sp.slot * a.H + h) * dg * vs;
  const int bank = reinterpret_cast<const PagedToken *>(blob + a.off_tokens)[sp.t0].bank;
  f4 st[P];
  auto load = [&](int c0, bool fresh) {
#pragma unroll
    for (int p = 0; p < P; ++p) {
      const int row = p * NG + rg;
      st[p] = f4{0.f, 0.f, 0.f, 0.f};
      if (!fresh && row < dg && c0 + cl < vs) st[p] = *reinterpret_cast<const f4 *>(S + (size_t)row * vs + c0 + cl);
    }
  };
  auto store = [&](int c0) {
#pragma unroll
    for (int p = 0; p < P; ++p) {
      const int row = p * NG + rg;
      if (row < dg && c0 + cl < vs) *reinterpret_cast<f4 *>(S + (size_t)row * vs + c0 + cl) = st[p];
    }
  };
  if (one) load(0, sp.pos0 == 0);
  float m = 0.f;
  if constexpr (RULE == kMemoryNormed)
    if (sp.pos0 > 0) m = a.peak[((size_t)sp.slot * 2 + bank) * a.H + h];

  const size_t slab = (size_t)a.T * a.y.NP, C = memory_columns(a);
  const int past = max(a.taps - 1, 0);
  const float *old = a.carry + ((size_t)sp.slot * 2 + bank) * past * C;
  float *now = a.carry + ((size_t)sp.slot * 2 + (bank ^ 1)) * past * C;
  // column c of q | k | v for token t of the span; keep: this workgroup carries it on
  auto project = [&](int t, int c, bool keep) {
    const size_t at = (size_t)(sp.t0 + t) * a.y.NP + a.col + c;
    const float u = sum_at(a.y, slab, at);
    float v = u;
    if (a.taps > 0) {
      if (keep) {
        const int ahead = sp.n - 1 - t;
        if (ahead < past) now[ahead * C + c] = u;
        if (t == 0)  // (a short span: earlier rows move on)
          for (int p = sp.n; p < past; ++p) now[p * C + c] = p - sp.n < sp.pos0 ? old[(p - sp.n) * C + c] : 0.f;
      }
      v = u * a.conv[past * C + c];
      for (int d = 1; d <= past && d <= sp.pos0 + t; ++d)
        v = fmaf(t >= d ? sum_at(a.y, slab, at - (size_t)d * a.y.NP) : old[(d - t - 1) * C + c],
                 a.conv[(past - d) * C + c], v);
    }
    return a.silu ? silu_f(v) : v;
  };
  int turn = 0;
  for (int p0 = 0; p0 < sp.n; p0 += piece) {
    const int np = min(piece, sp.n - p0);
    // the first product's columns
    {
      const int w = 2 * dg + vs;
      const bool first = h % (a.H / a.G) == 0;  // (query and key heads are shared)
      for (int id = tid; id < np * w; id += NT) {
        const int t = id / w, c = id - t * w;
        if (c < dg) sq[t * dg + c] = project(p0 + t, hq * dg + c, first);
        else if (c < 2 * dg) sk[t * dg + c - dg] = project(p0 + t, (a.G + hq) * dg + c - dg, first);
        else {
          const int vc = c - 2 * dg;
          float v = 0.f;
          if (vc < vg) v = project(p0 + t, 2 * a.G * dg + h * vg + vc, true);
          if (RULE == kMemoryNormed && vc == a.vdim) v = 1.f;
          sv[t * vs + vc] = v;
        }
      }
      const int r1 = a.decay.r, r2 = a.gate.r, rr = r1 + r2;
      for (int id = tid; id < np * rr; id += NT) {
        const int t = id / rr, c = id - t * rr;
        const float v = sum_at(a.y, slab, (size_t)(sp.t0 + p0 + t) * a.y.NP + (c < r1 ? a.decay.col + c : a.gate.col + c - r1));
        if (c < r1) sx[t * r1 + c] = v;
        else sx2[t * r2 + c - r1] = v;
      }
      if (tid < np) {
        const int t = sp.t0 + p0 + tid;
        if constexpr (RULE == kMemoryDelta)
          scal[tid * 8] = sigmoid_f(sum_at(a.y, slab, (size_t)t * a.y.NP + a.col_beta + h));
        if constexpr (RULE == kMemoryNormed) {
          float i, f;
          memory_gates(a, t, h, i, f);
          scal[tid * 8] = i, scal[tid * 8 + 1] = f;
        }
      }
    }
    __syncthreads();
    // gates, norms
    if constexpr (RULE == kMemoryNormed) {
      float mm = m, mine = 0.f;  // (every wave follows m for its own tokens)
      for (int t = 0; t < np; ++t) {
        const float i = scal[t * 8], f = scal[t * 8 + 1], mn = fmaxf(f + mm, i);
        if (t % NW == wave) {
          const float d = expf(f + mm - mn), kf = expf(i - mn);
          for (int c = lane; c < dg; c += 64) sg[t * dg + c] = d;
          if (lane == 0) scal[t * 8 + 3] = mn, scal[t * 8 + 4] = kf;
          mine = kf;
          for (int c = lane; c < dg; c += 64) {
            sq[t * dg + c] *= a.q_scale;
            sk[t * dg + c] *= mine;
          }
        }
        mm = mn;
      }
      m = mm;
    } else {
      for (int t = wave; t < np; t += NW) {
        float qq = 0.f, kk = 0.f, kq = 0.f;
        for (int c = lane; c < dg; c += 64) {
          const float x = sq[t * dg + c], y = sk[t * dg + c];
          qq = fmaf(x, x, qq), kk = fmaf(y, y, kk), kq = fmaf(x, y, kq);
        }
        float fq = a.q_scale, fk = 1.f;
        if (a.unit || RULE == kMemoryDelta) {
#pragma unroll
          for (int o = 32; o > 0; o >>= 1)
            qq += __shfl_xor(qq, o), kk += __shfl_xor(kk, o), kq += __shfl_xor(kq, o);
        }
        if (a.unit)
          fq *= __fdiv_rn(1.0f, sqrtf(qq + 1e-6f)), fk = __fdiv_rn(1.0f, sqrtf(kk + 1e-6f));
        for (int c = lane; c < dg; c += 64) {
          sq[t * dg + c] *= fq;
          sk[t * dg + c] *= fk;
        }
        if (lane == 0) scal[t * 8 + 2] = kq * fq * fk;
      }
      low_rank<E>(a.decay, h * a.dim, a.dim, np, sx,
                  [&](int t, int c, float z) { sg[t * dg + c] = expf(log_decay<RULE>(a, h, c, z)); });
      for (int id = tid; id < np * (dg - a.dim); id += NT)
        sg[id / (dg - a.dim) * dg + a.dim + id % (dg - a.dim)] = 1.f;
    }
    if (a.gate.r > 0) {
      low_rank<E>(a.gate, h * a.vdim, a.vdim, np, sx2, [&](int t, int c, float z) { sgate[t * vg + c] = z; });
      for (int id = tid; id < np * (vg - a.vdim); id += NT)
        sgate[id / (vg - a.vdim) * vg + a.vdim + id % (vg - a.vdim)] = 0.f;
    } else {
      for (int id = tid; id < np * vg; id += NT)
        sgate[id] = sum_at(a.y, slab, (size_t)(sp.t0 + p0 + id / vg) * a.y.NP + a.col_gate + h * vg + id % vg);
    }
    __syncthreads();
    // the tokens in turn
    for (int c0 = 0; c0 < vs; c0 += SW) {
      if (!one) load(c0, sp.pos0 + p0 == 0);
      const bool col = c0 + cl < vs;
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
          *reinterpret_cast<f4 *>(so + t * vs + c0 + cl) = o;
        }
      }
      if (!one || p0 + np >= sp.n) store(c0);
    }
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
      for (int c = lane; c < vg; c += 64) {
        const float gt = sgate[t * vg + c], w = a.norm[(a.norm_heads ? h * vg : 0) + c];
        const float v = c < a.vdim ? so[t * vs + c] * r * w * (a.gate_silu ? silu_f(gt) : sigmoid_f(gt)) : 0.f;
        const int oc = a.out_col + h * vg + c;
        st_elem((E *)a.out + (sizeof(E) == 2 ? act_packed_off(row, oc, a.ldo) : (size_t)row * a.ldo + oc), v);
      }
    }
    __syncthreads();
  }
  if constexpr (RULE == kMemoryNormed)
    if (tid == 0) a.peak[((size_t)sp.slot * 2 + (bank ^ 1)) * a.H + h] = m;
}

bool bad_shape(const Memory &a) {
  return a.H < 1 || a.G < 1 || a.H % a.G || a.dg % 32 || a.vg % 32 || a.dg < a.dim || a.vg < a.vdim ||
         a.dim < 1 || a.vdim < 1 || a.vs != memory_state_columns(a.rule, a.vdim) || a.vs < a.vg ||
         a.dg > kMemoryMaxDim || a.vs > kMemoryMaxVdim + 32 || a.y.S < 1 || a.y.S > 8 || a.y.NP % 4 || a.col % 4 ||
         a.taps < 0 || (a.taps > 0 && !a.conv) || (a.taps > 1 && !a.carry) || a.decay.r % 32 || a.gate.r % 32 ||
         (a.rule == kMemoryNormed ? !a.peak || !a.bi || !a.bf || a.decay.r : !a.decay.w || !a.dbias || !a.decay.r) ||
         (a.rule == kMemoryDelta && !a.rate) || !a.norm || !a.state || a.ldo % 32 || a.out_col % 32 ||
         a.out_col + a.H * a.vg > a.ldo;
}

template <MemoryRule RULE, class E>
hipError_t run_steps(const char *blob, int off_spans, int num_spans, const Memory &a, int limit, hipStream_t s) {
  // the widest power of two of columns that leaves at most 8 rows a thread
  int cw = 3;
  while (cw < 6 && (4 << cw) < a.vs && ((a.dg << (cw + 1)) + NT - 1) / NT <= 8) ++cw;
  const int rows = ((a.dg << cw) + NT - 1) / NT;
  const int red = 2 * 2 * NW * (4 << cw), each = piece_floats(a), budget = 16 * 1024;  // floats of LDS
  const int piece = std::min({kShortSpan, limit, std::max(1, (budget - red) / each)});
  const size_t bytes = (size_t)(red + piece * each) * 4;
  if (bytes > 64 * 1024) return hipErrorInvalidValue;
  const dim3 grid(a.H, num_spans);
#define FFMI_MS(P)                                                                                           \
  hipLaunchKernelGGL((memory_steps_kernel<RULE, E, P>), grid, dim3(NT), bytes, s, blob, off_spans, a, limit, \
                     piece, cw)
  if (rows <= 1) FFMI_MS(1);
  else if (rows <= 2) FFMI_MS(2);
  else if (rows <= 4) FFMI_MS(4);
  else if (rows <= 8) FFMI_MS(8);
  else return hipErrorInvalidValue;
#undef FFMI_MS
  return hipGetLastError();
}

}  // namespace

hipError_t launch_memory_steps(const char *blob, int off_spans, int num_spans, const Memory &a, bool f32,
                               int limit, hipStream_t s) {
  if (num_spans <= 0) return hipSuccess;
  if (bad_shape(a) || limit < 1) return hipErrorInvalidValue;
#define FFMI_MR(RULE)                                                                          \
  return f32 ? run_steps<RULE, float>(blob, off_spans, num_spans, a, limit, s)                 \
             : run_steps<RULE, uint16_t>(blob, off_spans, num_spans, a, limit, s)
  if (a.rule == kMemoryGated) FFMI_MR(kMemoryGated);
  if (a.rule == kMemoryDelta) FFMI_MR(kMemoryDelta);
  FFMI_MR(kMemoryNormed);
#undef FFMI_MR
}

}  // namespace ffmi
