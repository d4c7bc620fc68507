// latent.h -- latent attention over a paged cache (paged.h): launchers.
//
// A latent layer caches one vector c of `rank` elements per token, shared by
// every head (keys W_uk c, values W_uv c).  The kernels work in the absorbed
// form: q' = W_uk^T q per head, score = q' . c, o' = sum p c, out = W_uv o' --
// so all heads of a token are rows of one product against the same cache page.
#pragma once
#include "paged.h"

namespace ffmi {

// bf16 model: elements are bf16 bits, every width a multiple of 32, the rank a
// multiple of 64 that latent_rank_supported() accepts; fp32 model: floats.
bool latent_rank_supported(int rank);

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

}  // namespace ffmi
