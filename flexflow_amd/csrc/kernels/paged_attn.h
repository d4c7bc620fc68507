// paged_attn.h -- softmax attention with separate keys and values per head over
// a paged cache (paged.h): launchers.  Two kinds: scores with a bias by distance,
// and rotated queries and keys with soft-capped scores, windows and sinks.
//
// Query head h reads key/value head h / R (R = heads / groups).  Per layer the
// cache holds, page after page and in a page group after group, the MFMA
// operands of the two products:
//   keys    16 x 32 blocks of (key, dim), as packed activations: key_off
//   values  per 32 keys a row of those keys for every column, in the order the
//           score product leaves them in the lanes: val_off
#pragma once
#include <limits.h>

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
inline int attn_width(int dim) { return dim <= 64 ? 64 : dim <= 128 ? 128 : dim <= 256 ? 256 : 0; }

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
  // the rotary kind instead (no temperature, no mixing):
  //   q, k = rms_norm over the whole row of heads (y + b) * norms, norms [H dg | G dg]
  //   (null: y + b as it is), then columns 2m, 2m + 1 < rot turned by p * freq[m]
  //   turns and multiplied by rot_mult; v turned likewise by vfreq (null: not),
  //   [vg / 2]
  const double *freq = nullptr, *vfreq = nullptr;
  int rot = 0;
  float rot_mult = 1.f;
  // rotary kind, made in the attention's launch: taps > 0: a causal convolution of the
  // product's columns over time first (conv_rows.h; a launch of its own otherwise);
  // off_tokens: the step's tokens in its metadata
  const float *conv = nullptr;
  int taps = 0;
  float *carry = nullptr;
  int off_tokens = 0;
  bool unit = false;  // rotated queries and keys over their rms, per head
};
hipError_t launch_attn_prep(const char *blob, int off_tokens, int T, const AttnPrep &a, bool f32,
                            hipStream_t s);
hipError_t launch_rotary_prep(const char *blob, int off_tokens, int T, const AttnPrep &a, bool f32,
                              hipStream_t s);

// o[t][h] = softmax(q . k * scale + bias[h](distance)) v.  bias: per head D + 8
// floats, entry D + 3 - n for distance n (n from -4 to D + 3; D and above: the
// last row).  bf16: scale and bias for base-2 exponents, o in packed tiles of
// width H * vg; fp32: natural, o rows.
// The rotary kind: cap tanh(q . k * scale / cap) over the last `window` positions,
// exp(sink[h]) added to the softmax's denominator, values that were turned turned
// back by the query's position.
struct AttnArgs {
  const void *q = nullptr, *kc = nullptr, *vc = nullptr;
  const float *bias = nullptr;
  void *o = nullptr;
  int H = 0, G = 0, dp = 0, vg = 0, vp = 0, D = 0;
  float scale = 0.f;
  int ldo = 0;  // width of the rows that o is the first columns of (0: H * vg)
  // rotary kind.  cap_in: bf16 2 scale log2(e) / cap, fp32 scale / cap (0: no cap);
  // cap_out: cap (bf16: times log2(e)); sink: [H] (bf16: times log2(e)) or null;
  // off_tokens: the step's tokens in its metadata
  float cap_in = 0.f, cap_out = 0.f;
  int window = INT_MAX;
  const float *sink = nullptr;
  const double *vfreq = nullptr;
  int off_tokens = 0;
  float mult = 1.f;  // of the outputs
};
// bf16, widths that attn_width gave; slabs / ml: partials of split blocks, 16
// rows a slot, [slot][G][16][vp] and [slot][G][16][2].  pr: the launch makes
// queries, keys and values itself (launch_attn_prep's work; a.q is not read) --
// steps whose blocks have at most 16 rows only (pl.row_tiles == 1)
hipError_t launch_paged_attn(const char *blob, const PagedLists &pl, const AttnArgs &a, float *slabs,
                             float *ml, hipStream_t s, const AttnPrep *pr = nullptr, int T = 0);
hipError_t launch_rotary_attn(const char *blob, const PagedLists &pl, const AttnArgs &a, float *slabs,
                              float *ml, hipStream_t s, const AttnPrep *pr = nullptr, int T = 0);
constexpr int kAttnTiles = 4;  // row tiles of a workgroup in prompts
// any width up to kAttnRowsMax, one workgroup per row of every block (fp32, or
// bf16 with scale and bias for base-2 exponents as above)
constexpr int kAttnRowsMax = 1024;
hipError_t launch_paged_attn_rows(const char *blob, const PagedLists &pl, const AttnArgs &a, bool f32,
                                  hipStream_t s);
hipError_t launch_rotary_attn_rows(const char *blob, const PagedLists &pl, const AttnArgs &a, bool f32,
                                   hipStream_t s);

}  // namespace ffmi
