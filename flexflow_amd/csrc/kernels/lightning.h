// lightning.h -- linear attention with a fixed decay per head: launchers.
//
// Per head S_t = d S_(t-1) + k_t v_t^T, o_t = S_t^T q_t with q, k, v = silu of
// their projections.  The state S [dim][vdim] is fp32, one per request slot:
// [slots][H][dg][vg], read and written by the steps that bring the request's
// tokens; position 0 starts from zeros.
//
// Projections y: sums of one product, columns q [H][dg] | k [H][dg] | v [H][vg] |
// gate [H][vg] (dg, vg: dim, vdim in whole 32-column steps, zero beyond).
#pragma once
#include "paged.h"

namespace ffmi {

struct Lightning {
  Partials y;
  const float *powers = nullptr;  // [H][kLightningChunk + 1]: d^0, d^1, ...
  float *state = nullptr;
  uint16_t *qkv = nullptr;  // bf16 [T][2 H dg + H vg], for the chunked form
  float *o = nullptr;       // [T][H vg]
  int H = 0, dg = 0, vg = 0, T = 0;
};
constexpr int kLightningChunk = 64;
constexpr int kLightningMaxDim = 512;        // token-by-token form
constexpr int kLightningMaxChunkDim = 256;   // chunked form

// token by token: spans of at most `limit` tokens
hipError_t launch_lightning_recurrent(const char *blob, int off_spans, int num_spans,
                                      const Lightning &a, int limit, hipStream_t s);
// chunks of 64 tokens on MFMA: spans of more than `limit` tokens.  Decays and
// the state stay fp32: what meets a product besides q, k, v goes in as two bf16
// terms (value and remainder).
hipError_t launch_lightning_chunks(const char *blob, int off_spans, int num_spans, const Lightning &a,
                                   int limit, hipStream_t s);
// out = o / rms(o) * w * sigmoid(gate) over all heads together (n real columns
// of H vg): bf16 packed tiles (hb) or fp32 rows (hf)
hipError_t launch_gated_norm(const float *o, const Partials &y, int gate_col, const float *w,
                             uint16_t *hb, float *hf, int T, int H, int n, float eps, hipStream_t s);

}  // namespace ffmi
