// latent.h -- latent attention over a paged cache: step metadata and launchers.
//
// A latent layer caches one vector c of `rank` elements per token, shared by
// every head (keys W_uk c, values W_uv c).  The kernels work in the absorbed
// form: q' = W_uk^T q per head, score = q' . c, o' = sum p c, out = W_uv o' --
// so all heads of a token are rows of one product against the same cache page.
//
// The cache is a pool of pages of kPageTokens tokens; a request's page table
// lists the pages of its positions in order.
#pragma once
#include "../ffmi_internal.h"

namespace ffmi {

constexpr int kPageTokens = 64;

struct PagedToken {
  int32_t token, pos;  // embedding row, position in the sequence
  int32_t row;         // cache row: page * kPageTokens + offset
  int32_t pad;
};

// One workgroup of the attention: `nrows` consecutive (token, head) rows of a
// request (row = batch token * heads + head) against cache tiles (= pages)
// [tile0, tile0 + ntiles).  slot >= 0: a partial result for a LatentMerge.
struct LatentBlock {
  int32_t row0, nrows;   // nrows == 0: padding, nothing to do
  int32_t seg_row, pos0;  // first row of the request's tokens, its position
  int32_t table;          // offset of the request's page table (int32 units)
  int32_t tile0, ntiles;
  int32_t slot;
  int32_t page0;          // the page of tile0: one dependent load less at the start
  int32_t pad[3];
};
struct LatentMerge {
  int32_t row0, nrows, slot0, nslots;
};

// Layout of a step's metadata, packed by runtime/paged_step.cpp.  Offsets in
// bytes from the start of the blob.
struct PagedLists {  // the block lists of the layers with one head count
  int heads = 0, row_tiles = 0;  // rows per block / 16
  int num_blocks = 0, num_merges = 0, off_blocks = 0, off_merges = 0;
};

// bf16 model: elements are bf16 bits, every width a multiple of 32, the rank a
// multiple of 64 that latent_rank_supported() accepts; fp32 model: floats.
bool latent_rank_supported(int rank);

// x = embed[token] + pos[p] in fp32; xb (optional) the bf16 packed tiles.
// blob_src: the step's staging in mapped host memory, copied to blob_dst by
// this first kernel of the step.
hipError_t launch_embed_pos(const char *blob_src, char *blob_dst, size_t blob_bytes,
                            const uint16_t *embed, const uint16_t *pos, float *x, uint16_t *xb,
                            int T, int H, hipStream_t s);
// x += y / rms(y) * w on n columns (row stride H); y = sum of the fp32 slabs;
// xb (optional): the new x in bf16 packed tiles
hipError_t launch_post_norm(Partials y, const float *w, float *x, uint16_t *xb, int T, int H, int n,
                            float eps, hipStream_t s);
// h[i] = x[rows[i]] / rms * w: bf16 packed tiles (hb) or fp32 rows (hf)
hipError_t launch_row_norm(const char *blob, int off_rows, const float *x, const float *w,
                           uint16_t *hb, float *hf, int R, int H, int n, float eps, hipStream_t s);
hipError_t launch_relu2_f32(float *u, size_t n, hipStream_t s);

// Per-head products Y[t][h] = X[t][h] . W_h^T (+ sigmoid gate).  X: row stride
// ldx, head stride kh; gate: pre-activation [T][ldg] (null: none).
struct HeadGemm {
  const void *X = nullptr, *W = nullptr, *gate = nullptr;
  void *Y = nullptr;
  int T = 0, heads = 0, K = 0, N = 0, ldx = 0, ldg = 0;
  bool packed = false;  // bf16: Y in packed activation tiles of width heads * N
};
// Normed latent rows to the cache: c = d / rms(d) * w over n of `rank` columns
struct LatentStore {
  const void *d = nullptr;  // [T][ldd], this layer's down-projection columns
  const float *w = nullptr;
  void *cache = nullptr;
  int ldd = 0, rank = 0, n = 0;
  float eps = 0.f;
};
// bf16: one launch runs the store's and the product's workgroups together
// (st.cache == null: no store, a layer that reads another layer's cache)
hipError_t launch_latent_prep(const char *blob, int off_tokens, const LatentStore &st,
                              const HeadGemm &hg, hipStream_t s);
hipError_t launch_head_gemm(const HeadGemm &hg, hipStream_t s);
hipError_t launch_latent_store_f32(const char *blob, int off_tokens, int T, const LatentStore &st,
                                   hipStream_t s);
hipError_t launch_head_gemm_f32(const HeadGemm &hg, hipStream_t s);

// o[row] = softmax(q'[row] . c * scale) c over the row's visible positions;
// q, o [T * heads][rank]; slabs / ml: partials of split blocks
hipError_t launch_latent_attention(const char *blob, const PagedLists &pl, const uint16_t *q,
                                   const uint16_t *cache, uint16_t *o, float *slabs, float *ml,
                                   int rank, float scale, hipStream_t s);
// any rank, one workgroup per row of every block (element: fp32, or bf16 when
// the rank has no MFMA form)
hipError_t launch_latent_attention_rows(const char *blob, const PagedLists &pl, const void *q,
                                        const void *cache, void *o, int rank, float scale,
                                        bool bf16, hipStream_t s);

// dst = the [N][K] matrix a kernel wants, from the checkpoint's src: row n =
// head n / np's row n % np (zero from nb on; heads * np rows), column k
// likewise from (kb, kp).  transpose: src holds [heads][K][N] blocks.
// perhead: each head its own tile-major packed block (head products).
struct PackSpec {
  int rows = 0, nb = 0, np = 0;  // heads, real rows per head, padded rows per head
  int cols = 0, kb = 0, kp = 0;
  bool transpose = false;
};
hipError_t launch_pack_bf16(const uint16_t *src, int ld, const PackSpec &p, uint16_t *dst,
                            int tile_offset, int pitch, bool perhead, hipStream_t s);
// row-major [T][K] bf16 -> packed activation tiles (rows past T zero)
hipError_t launch_pack_act_bf16(const uint16_t *X, uint16_t *Xp, int T, int K, hipStream_t s);
hipError_t launch_pack_f32(const uint16_t *src, int ld, const PackSpec &p, float *dst,
                           hipStream_t s);

}  // namespace ffmi
