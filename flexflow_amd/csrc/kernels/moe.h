// moe.h -- mixture of experts: routing, row lists, products by expert: launchers
// (moe.hip).
//
// A token's chosen experts are rows ("slots") of products grouped by expert: every
// expert's slots lie together, from a multiple of 16 on.  A shared expert that runs
// for every token joins the first product as one more group, its slots the tokens in
// order; its units, times the token's gate, are columns of a wider activation, so
// that its second product is part of a dense one.
#pragma once
#include "../ffmi_internal.h"

namespace ffmi {

struct MoeTile {
  int32_t expert;  // == number of experts: the shared one
  int32_t slot0, rows, pad;
};
constexpr int kMoeFew = 16, kMoeMany = 256;  // rows of a tile in the two forms
constexpr int kMoeMaxExperts = 1024, kMoeMaxTop = 64;

// a step's sizes: T tokens of which each takes `top` of `experts`
struct MoeSizes {
  int T = 0, experts = 0, top = 0;
  int identity = 0;  // further outputs of the router, after the experts': the row itself
  bool shared = false;
  int gate_col = 0;  // column of the shared expert's gate in the router's product
  int tile_rows() const {
    return T > 32 && (long)T * top >= 4L * experts ? kMoeMany : kMoeFew;
  }
  // upper bounds: slots of the experts (whole 16s), tiles
  __host__ __device__ int slots() const {
    const int a = T * top, e = a < experts ? a : experts;
    return (a + 15 * e + 15) / 16 * 16;
  }
  int expert_tiles(int rows) const {
    const int a = T * top, e = a < experts ? a : experts;
    return (a - e) / rows + e;
  }
  __host__ __device__ int shared_tiles(int rows) const { return shared ? (T + rows - 1) / rows : 0; }
};
struct MoeLists {
  int32_t *picked = nullptr;      // [T][top] experts
  int32_t *at = nullptr;          // [T][top] slots (-1: none, an identity expert)
  float *wt = nullptr;            // [T][top] their weights
  float *gate = nullptr;          // [T] the shared expert's
  float *own = nullptr;           // [T] the identity experts' weights together
  int32_t *slot_token = nullptr;  // [slots]
  MoeTile *tiles = nullptr;       // the shared expert's first
  int32_t *num_tiles = nullptr;
};
// z: router products, the experts' columns first.  The `top` largest z + bias (the
// lowest index among equals), softmax over them; gate: the sigmoid of its column.
hipError_t launch_moe_route(const Partials &z, const float *bias, const MoeSizes &n, const MoeLists &l,
                            hipStream_t s);
// Another choice: scores s = softmax of all columns (identity experts' included); the
// `top` largest s + correction among the columns of the best `keep` of `groups` equal
// groups of neighbours (a group counts as its best column); weights scale s / (sum of
// the chosen s + 1e-20).
struct MoeScores {
  const float *correction = nullptr;  // [experts + identity]
  int groups = 1, keep = 1;
  float scale = 1.f;
};
hipError_t launch_moe_route_scores(const Partials &z, const MoeScores &sc, const MoeSizes &n, const MoeLists &l,
                                   hipStream_t s);

// One product of every slot with its expert's matrix.
//   first  (gated): Y[slot] = silu(X W_gate) (X W_up), X the token's row (row-major),
//          Y bf16 in packed tiles of width ldy (fp32: rows); the shared expert's
//          times gate[token].  limit > 0: the clamped gated unit instead
//   second: Y[slot] = X W_down, X the first product's Y; Y rows of N, bf16 (fp32)
// W: bf16 packed weights, gate / up tiles in turn (fp32: rows, gate then up), expert
// after expert.
struct MoeGroup {
  const void *X = nullptr, *W = nullptr;
  void *Y = nullptr;
  int N = 0, K = 0, ldy = 0;
  size_t w_stride = 0;  // elements from expert to expert
};
struct MoeGemm {
  MoeGroup g[2];  // experts, shared (first product)
  int experts = 0;
  const int32_t *slot_token = nullptr;
  const MoeTile *tiles = nullptr;
  const int32_t *num_tiles = nullptr;
  const float *gate = nullptr;
  float limit = 0.f;
};
hipError_t launch_moe_gemm(const MoeGemm &a, const MoeSizes &n, bool gated, bool f32, bool stream_weights,
                           hipStream_t s);

}  // namespace ffmi
