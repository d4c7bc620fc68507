// conv_rows.h -- a short causal convolution over time of a product's columns: launcher
// (conv_rows.hip).
//
// y_t = sum over j < taps of conv[j] u_(t - taps + 1 + j), u the columns [col, col + cols)
// of deferred sums, zeros before the sequence.  The last taps - 1 rows u of a request are
// carried from step to step: carry [slots][2 banks][taps - 1][cols], the latest first; a
// step reads one bank and writes the other.
#pragma once
#include "paged.h"

namespace ffmi {

struct ConvRows {
  Partials u;
  int T = 0, col = 0, cols = 0;
  int taps = 0;
  const float *conv = nullptr;  // [taps][cols], the last row the current token's
  float *carry = nullptr;
  bool silu = false;  // of y
  // [T][cols], bf16 or fp32
  uint16_t *hb = nullptr;
  float *hf = nullptr;
  int off_tokens = 0;
  int above = 0;  // only tokens of portions of more than so many tokens
};
hipError_t launch_conv_rows(const char *blob, const ConvRows &a, hipStream_t s);

}  // namespace ffmi
