// conv_norm.h -- the 32-bit residual stream of parallel layers with a causal
// convolution at the mixer's input: launchers (conv_norm.hip).
#pragma once
#include "residual.h"

namespace ffmi {

// x = x_in + mult * (sum of y's slabs + sum over k of wt[t][k] rows[at[t][k]])
// h = x in `groups` equal parts, each over its own rms, times w
// c = h + sum over j < taps of conv[j] h_(t - taps + 1 + j)
// The last taps - 1 rows h of a request are carried from step to step: `carry`
// [slots][2 banks][taps - 1][H], the latest first.  Rows are H floats, the first
// n of them real.
struct ConvNorm {
  Partials y;  // S == 0: none
  const void *rows = nullptr;  // null: none; bf16 or (rows_f32) fp32, [.][H]
  const int32_t *at = nullptr;
  const float *wt = nullptr;
  int top = 0;
  bool rows_f32 = false;
  const float *x_in = nullptr;
  float *x = nullptr;  // another buffer than x_in (null: not wanted)
  float mult = 1.f;
  const float *w = nullptr;  // null: the sum only
  int H = 0, n = 0, groups = 1;
  float eps = 0.f;
  const float *conv = nullptr;  // [taps][H]; null: no convolution
  int taps = 0;
  float *carry = nullptr;
  float *inv = nullptr;  // [T][groups] scratch (convolution): 1 / rms of the groups
  // h and c in packed tiles, rows of bf16, or rows of fp32 (null: not wanted)
  uint16_t *hb = nullptr, *hrow = nullptr, *cb = nullptr;
  float *hf = nullptr, *cf = nullptr;
};
// Where the rows x come from in the first layer: embed[token] * scale, plus (with a
// table of buckets + 1 rows) pairs[(prev mul_prev + token mul_cur) mod buckets], the
// last row where no token is before.
struct EmbedPairs {
  const uint16_t *embed = nullptr, *pairs = nullptr;
  float scale = 1.f;
  int buckets = 0;
  int64_t mul_prev = 0, mul_cur = 0;
};

// every token of the step.  em: the step's first kernel, which also copies the
// staging blob_src (mapped host memory, tokens first) to blob_dst; else blob_src
// is the device copy
hipError_t launch_conv_norm(const char *blob_src, char *blob_dst, size_t blob_bytes, int off_tokens,
                            const ConvNorm &a, const EmbedPairs *em, int T, hipStream_t s);
// h of the listed rows, in their order (no convolution, x not kept)
hipError_t launch_conv_norm_rows(const char *blob, int off_tokens, int off_rows, const ConvNorm &a, int T,
                                 int R, hipStream_t s);

}  // namespace ffmi
