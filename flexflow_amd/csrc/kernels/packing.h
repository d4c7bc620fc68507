// packing.h -- weight and activation layouts: launchers (packing.hip).
#pragma once
#include "../ffmi_internal.h"

namespace ffmi {

// dst = the [N][K] matrix a kernel wants, from the checkpoint's src: row n =
// head n / np's row n % np (zero from nb on; heads * np rows), column k
// likewise from (kb, kp).  transpose: src holds [heads][cols][kb][N] blocks.
// plus: added to every element that is not padding (pack_f32).
// perhead: each head its own tile-major packed block (head products).
// row_pairs / col_pairs: of every head's first so many rows (columns), m and
// m + half of them come to lie side by side (rotations that pair halves).
// k0 / kt: the matrix is k-steps k0 .. of a destination of kt k-steps, 32
// columns each (0: the destination is this matrix alone).
struct PackSpec {
  int rows = 0, nb = 0, np = 0;  // heads, real rows per head, padded rows per head
  int cols = 0, kb = 0, kp = 0;
  bool transpose = false;
  int row_pairs = 0, col_pairs = 0;
  int k0 = 0, kt = 0;
  float plus = 0.f;
};
hipError_t launch_pack_bf16(const uint16_t *src, int ld, const PackSpec &p, uint16_t *dst,
                            int tile_offset, int pitch, bool perhead, hipStream_t s,
                            int tile_step = 1);
// row-major [T][K] bf16 -> packed activation tiles (rows past T zero)
hipError_t launch_pack_act_bf16(const uint16_t *X, uint16_t *Xp, int T, int K, hipStream_t s);
hipError_t launch_pack_f32(const uint16_t *src, int ld, const PackSpec &p, float *dst,
                           hipStream_t s);

}  // namespace ffmi
