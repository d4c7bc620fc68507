// residual.h -- the 32-bit residual stream: launchers (residual.hip).
#pragma once
#include "paged.h"

namespace ffmi {

// x = embed[token] + pos[p] (pos null: the embedding alone) in fp32; xb (optional) the
// bf16 packed tiles.
// blob_src: the step's staging in mapped host memory, copied to blob_dst by
// this first kernel of the step.
hipError_t launch_embed_pos(const char *blob_src, char *blob_dst, size_t blob_bytes,
                            const uint16_t *embed, const uint16_t *pos, float *x, uint16_t *xb,
                            int T, int H, hipStream_t s);
// x = embed[token] * scale in fp32, h = x / rms(x) * w as launch_add_norm's; the
// first kernel of a step, as above
hipError_t launch_embed_norm(const char *blob_src, char *blob_dst, size_t blob_bytes,
                             const uint16_t *embed, float scale, const float *w, float *x,
                             uint16_t *hb, float *hf, int T, int H, int n, float eps, hipStream_t s);
// x += y / rms(y) * w on n columns (row stride H); y = sum of the fp32 slabs;
// xb (optional): the new x in bf16 packed tiles
hipError_t launch_post_norm(Partials y, const float *w, float *x, uint16_t *xb, int T, int H, int n,
                            float eps, hipStream_t s);
// x += y (y.S == 0: nothing to add), h = x / rms(x) * w: bf16 packed tiles (hb)
// or fp32 rows (hf); w null: the sum only
hipError_t launch_add_norm(Partials y, const float *w, float *x, uint16_t *hb, float *hf, int T,
                           int H, int n, float eps, hipStream_t s);
// h[i] = x[rows[i]] / rms * w: bf16 packed tiles (hb) or fp32 rows (hf)
hipError_t launch_row_norm(const char *blob, int off_rows, const float *x, const float *w,
                           uint16_t *hb, float *hf, int R, int H, int n, float eps, hipStream_t s);
// The stream normed after every sum:
//   x = norm(alpha x + sum of y's slabs + sum over k of wt[t][k] rows[at[t][k]]
//            + own[t] x) w
// rows (of experts; at < 0: none): bf16 or (rows_f32) fp32, [.][H].  Besides x: bf16
// packed tiles (hb) and bf16 rows (hrow) of it.
struct SumNorm {
  Partials y;  // S == 0: none
  const void *rows = nullptr;
  bool rows_f32 = false;
  const int32_t *at = nullptr;
  const float *wt = nullptr, *own = nullptr;
  int top = 0;
  float alpha = 1.f, eps = 0.f;
  const float *w = nullptr;
  float *x = nullptr;
  uint16_t *hb = nullptr, *hrow = nullptr;
  int T = 0, H = 0, n = 0;  // columns, the first n of them real
};
hipError_t launch_sum_norm(const SumNorm &a, hipStream_t s);
// packed bf16 rows of the columns [col, col + n) of deferred sums, n a multiple of 32
hipError_t launch_pack_sums(const Partials &y, int col, uint16_t *out, int T, int n, hipStream_t s);
hipError_t launch_relu2_f32(float *u, size_t n, hipStream_t s);
// Y[T][F] = clamped_glu of gu [T][gate F | up F]
hipError_t launch_glu_f32(const float *gu, float *Y, int T, int F, float limit, hipStream_t s);
// the same with a SiLU gate, Y rows of ldy
hipError_t launch_swiglu_f32(const float *gu, float *Y, int T, int F, int ldy, hipStream_t s);
// z = cap tanh(z / cap) on n columns of rows of ld
hipError_t launch_soft_cap(float *z, int R, int n, int ld, float cap, hipStream_t s);

}  // namespace ffmi
