// paged_attn.h -- softmax attention with separate keys and values per head over
// a paged cache (paged.h), with a bias by distance: launchers.
//
// Query head h reads key/value head h / R (R = heads / groups).  Per layer the
// cache holds, page after page and in a page group after group, the MFMA
// operands of the two products:
//   keys    16 x 32 blocks of (key, dim), as packed activations: key_off
//   values  per 32 keys a row of those keys for every column, in the order the
//           score product leaves them in the lanes: val_off
#pragma once
#include "paged.h"

namespace ffmi {

// element (key 0..63, column c < dp) / (column c < vp, key) of a group's page
__host__ __device__ __forceinline__ int key_off(int key, int c, int dp) {
  return (((key >> 4) * (dp >> 5) + (c >> 5)) * 64 + (key & 15) + 16 * ((c >> 3) & 3)) * 8 + (c & 7);
}
__host__ __device__ __forceinline__ int val_off(int key, int c, int vp) {
  const int k = key & 31;
  return ((key >> 5) * vp + c) * 32 + ((k & 15) >> 2) * 8 + (k & 3) + 4 * (k >> 4);
}
// cache widths of the bf16 form (0: none, the row form takes the width as it is)
int attn_width(int dim);

// Queries, keys and values from the sums y of their product (columns q [H][dg] |
// k [G][dg] | v [G][vg]):
//   q = rms_norm(y + b) * w * (1 + coef ln((p + 1) / every + 1))  -> q [T][H][dp]
//   k = rms_norm(y + b) * w                                       -> cache
//   v = y + b; v = (1 - mix) v + mix first                        -> cache
struct AttnPrep {
  Partials y;
  const float *bias = nullptr;                    // [columns]
  const float *norms = nullptr;                   // [dg] of the queries, [dg] of the keys
  const float *vmix = nullptr;  // null: v as it is
  float *first = nullptr;       // values [T][G][vg]: written (vmix null) or read
  void *q = nullptr, *kc = nullptr, *vc = nullptr;
  int H = 0, G = 0, dim = 0, dg = 0, dp = 0, vg = 0, vp = 0;
  float eps = 0.f, coef = 0.f;  // coef 0: no temperature
  int every = 1;
};
hipError_t launch_attn_prep(const char *blob, int off_tokens, int T, const AttnPrep &a, bool f32,
                            hipStream_t s);

// o[t][h] = softmax(q . k * scale + bias[h](distance)) v.  bias: per head D + 8
// floats, entry D + 3 - n for distance n (n from -4 to D + 3; D and above: the
// last row).  bf16: scale and bias for base-2 exponents, o in packed tiles of
// width H * vg; fp32: natural, o rows.
struct AttnArgs {
  const void *q = nullptr, *kc = nullptr, *vc = nullptr;
  const float *bias = nullptr;
  void *o = nullptr;
  int H = 0, G = 0, dp = 0, vg = 0, vp = 0, D = 0;
  float scale = 0.f;
};
// bf16, widths that attn_width gave; slabs / ml: partials of split blocks, 16
// rows a slot, [slot][G][16][vp] and [slot][G][16][2].  pr: the launch makes
// queries, keys and values itself (launch_attn_prep's work; a.q is not read) --
// steps whose blocks have at most 16 rows only (pl.row_tiles == 1)
hipError_t launch_paged_attn(const char *blob, const PagedLists &pl, const AttnArgs &a, float *slabs,
                             float *ml, hipStream_t s, const AttnPrep *pr = nullptr, int T = 0);
constexpr int kAttnTiles = 4;  // row tiles of a workgroup in prompts
// any width up to kAttnRowsMax, one workgroup per row of every block (fp32, or
// bf16 with scale and bias for base-2 exponents as above)
constexpr int kAttnRowsMax = 1024;
hipError_t launch_paged_attn_rows(const char *blob, const PagedLists &pl, const AttnArgs &a, bool f32,
                                  hipStream_t s);

}  // namespace ffmi
