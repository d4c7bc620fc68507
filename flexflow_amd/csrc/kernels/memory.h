// memory.h -- matrix memories: linear attention whose state S [dim][vdim] (fp32, one per
// request slot and head) forgets by gates that the tokens themselves give: launchers
// (memory.hip: token by token; memory_chunks.hip: chunks of 64 tokens on MFMA).
//
//   gated   S = diag(g) S + k v^T                       o = S^T q
//   delta   S = diag(g) S;  u = beta (v - S^T k);  S += k u^T   o = S^T q
//   normed  S = d S + w k v^T, n likewise with 1 in v's place, gates exp(.) kept in range
//           by a running maximum m (it starts at 0):
//           m' = max(f + m, i), d = exp(f + m - m'), w = exp(i - m')
//           o = S^T q / (max(|n . q|, exp(-m)) + 1e-6)
//
// g, per head and key channel: sigmoid(z)^(1 / tau) (gated) or exp(-rate softplus(z))
// (delta), z = A2 (A1 h) + bias, a product through few columns (LowRank).  i and f, per
// head: i = cap tanh((W_i h + b) / cap), f = logsigmoid(cap tanh((W_f h + b) / cap)).
// Then every head's o over its rms, times a weight, times a gate: sigmoid or SiLU of
// columns of the first product or of another LowRank.
#pragma once
#include "paged.h"

namespace ffmi {

enum MemoryRule { kMemoryGated, kMemoryDelta, kMemoryNormed };

// Columns of the first product times a second, narrow matrix.
struct LowRank {
  int col = 0, r = 0;       // columns [col, col + r) of the first product (r: whole 32s)
  const void *w = nullptr;  // rows [outputs][r], bf16 (fp32 model: fp32)
  int zcol = 0;             // the outputs' first column in Memory::z
};

struct Memory {
  MemoryRule rule = kMemoryGated;
  // query / key heads, heads; real and padded widths; columns of the state (vg; normed:
  // at least vdim + 1, the column vdim is n)
  int T = 0, G = 0, H = 0, dim = 0, dg = 0, vdim = 0, vg = 0, vs = 0;
  // sums of the first product: q [G][dg] | k [G][dg] | v [H][vg] from column `col` on
  Partials y;
  int col = 0;
  // taps > 0: a causal convolution of those columns over time; conv [taps][columns], the
  // last row the current token's; carried rows [slots][2 banks][taps - 1][columns], the
  // latest first
  int taps = 0;
  const float *conv = nullptr;
  float *carry = nullptr;
  bool silu = false;  // then SiLU
  bool unit = false;  // then q and k over sqrt(sum of squares + 1e-6), per head
  float q_scale = 1.f;
  // gates
  LowRank decay;
  const float *dbias = nullptr;  // [H dg]
  const float *rate = nullptr;   // delta: [H]
  float inv_tau = 1.f;           // gated
  int col_beta = 0;              // delta: [H] columns, before their sigmoid
  int col_i = 0, col_f = 0;      // normed: [H] columns each
  const float *bi = nullptr, *bf = nullptr;
  float cap = 1.f;
  Partials z;  // chunks: sums of the second products
  float *state = nullptr;  // [slots][H][dg][vs]
  float *peak = nullptr;   // normed: m, [slots][2 banks][H]
  // outputs: columns [out_col, out_col + H vg) of rows of ldo, bf16 packed tiles or fp32
  const float *norm = nullptr;  // [vg], or [H][vg] (norm_heads)
  bool norm_heads = false;
  float eps = 0.f;
  bool gate_silu = false;
  int col_gate = 0;  // the gate's [H vg] columns of the first product ...
  LowRank gate;      // ... or (r > 0) a second one's
  void *out = nullptr;
  int ldo = 0, out_col = 0;
  int off_tokens = 0;  // the step's tokens in its metadata
};
constexpr int kMemoryChunk = kSpanChunk;
constexpr int kMemoryMaxDim = 512, kMemoryMaxVdim = 2048;  // token by token
constexpr int kMemoryMaxChunkDim = 256;                    // chunks
inline int memory_state_columns(MemoryRule r, int vdim) {
  return (vdim + (r == kMemoryNormed) + 31) / 32 * 32;
}

// Scratch, from the step's bounds: per (chunk, head) the operands of the pass over the
// chunks, per token what the launches after it take.
struct MemoryScratch {
  uint16_t *rows = nullptr;                             // delta: [T][columns of q | k | v]
  uint16_t *qg = nullptr, *kd = nullptr, *w = nullptr;  // [64][DK], [DK][64], [64][DK] (delta)
  uint16_t *p = nullptr;                                // [64][64]
  float *u = nullptr;                                   // delta: [64][vs]
  float *last = nullptr;                                // [DK]
  float *gates = nullptr;                               // normed: [T][H][3]
  float *o = nullptr;                                   // [T][H][vs]
};
inline int memory_chunk_width(int dg) { return dg <= 32 ? 32 : dg <= 64 ? 64 : dg <= 128 ? 128 : 256; }
// most chunks that a step of T tokens in so many spans has
inline size_t memory_chunks_max(int T, int spans) { return (size_t)T / kMemoryChunk + spans; }

// Token by token: spans of at most `limit` tokens, everything in one launch, unless the
// heads are few and wide: with scratch (w) their columns are then split, the outputs are
// left in w.o (*left) and launch_memory_out has to follow.
hipError_t launch_memory_steps(const char *blob, int off_spans, int num_spans, const Memory &a,
                               const MemoryScratch *w, bool f32, int limit, bool *left, hipStream_t s);
// Chunks (bf16 model): spans of more than `limit` >= kShortSpan tokens; num_chunks: the
// step's (PagedSpan::chunk0 counts them).  The outputs are left in w.o.
hipError_t launch_memory_chunks(const char *blob, int off_spans, int num_spans, int num_chunks, const Memory &a,
                                const MemoryScratch &w, int limit, hipStream_t s);
// norm and gate of w.o, for the tokens of spans of more than `above` tokens
hipError_t launch_memory_out(const char *blob, const Memory &a, const MemoryScratch &w, int above, hipStream_t s);

}  // namespace ffmi
