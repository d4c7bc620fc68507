// capi_latent.cpp -- C ABI of the bf16 products and latent attention
// (include/ffmi.h): one operator at a time, for callers outside the models.
#include <algorithm>
#include <vector>

#include "../kernels/latent.h"
#include "../kernels/packing.h"
#include "../kernels/residual.h"
#include "device_buf.h"
#include "paged_step.h"

extern "C" ffmi_status ffmi_linear_bf16(const void *X, const void *W, void *Y, int T, int out_dim,
                                        int in_dim, int epilogue, ffmi_stream stream) {
  using namespace ffmi;
  FFMI_CHECK(X && W && Y && T > 0 && out_dim > 0 && in_dim > 0, FFMI_ERR_INVALID);
  FFMI_CHECK(out_dim % 32 == 0 && in_dim % 32 == 0, FFMI_ERR_UNSUPPORTED);
  FFMI_CHECK(epilogue >= FFMI_BF16_PLAIN && epilogue <= FFMI_BF16_SUM, FFMI_ERR_INVALID);
  hipStream_t s = (hipStream_t)stream;
  const size_t wsb = gemm_bf16_workspace_bytes(T, out_dim, in_dim);
  DeviceBuf xp, wp, ws;
  const size_t xbytes = (size_t)((T + 15) / 16) * 16 * in_dim * 2;
  if (!xp.get(xbytes) || !wp.get((size_t)out_dim * in_dim * 2) || !ws.get(wsb)) return FFMI_ERR_OOM;
  FFMI_HIP(launch_pack_act_bf16((const uint16_t *)X, (uint16_t *)xp.p, T, in_dim, s));
  PackSpec p;
  p.rows = p.cols = 1, p.nb = p.np = out_dim, p.kb = p.kp = in_dim;
  FFMI_HIP(launch_pack_bf16((const uint16_t *)W, in_dim, p, (uint16_t *)wp.p, 0, out_dim / 16,
                            false, s));
  const uint16_t *x = (const uint16_t *)xp.p, *w = (const uint16_t *)wp.p;
  float *wsp = (float *)ws.p;
  if (epilogue == FFMI_BF16_PLAIN)
    FFMI_HIP(launch_gemm_bf16_plain(x, w, (uint16_t *)Y, wsp, wsb, T, out_dim, in_dim, FFMI_X_PACKED, s));
  else if (epilogue == FFMI_BF16_RELU2)
    FFMI_HIP(launch_gemm_bf16_relu2(x, w, (uint16_t *)Y, wsp, wsb, T, out_dim, in_dim, FFMI_X_PACKED, s));
  else
    FFMI_HIP(launch_gemm_bf16_f32(x, w, nullptr, (float *)Y, (size_t)T * out_dim * 4, T, out_dim,
                                  in_dim, FFMI_X_PACKED, s));
  FFMI_HIP(hipStreamSynchronize(s));  // (the packed operands are freed here)
  return FFMI_OK;
}

extern "C" ffmi_status ffmi_post_rmsnorm(const float *y, int slabs, const float *w, float *x, int T,
                                         int H, int n, float eps, ffmi_stream stream) {
  FFMI_CHECK(y && w && x && T > 0 && H > 0 && n > 0 && n <= H && slabs >= 1 && slabs <= 8,
             FFMI_ERR_INVALID);
  FFMI_CHECK(H % 32 == 0 && H <= 16384, FFMI_ERR_UNSUPPORTED);
  ffmi::Partials p;
  p.p = y, p.S = slabs, p.NP = H;
  FFMI_HIP(ffmi::launch_post_norm(p, w, x, nullptr, T, H, n, eps, (hipStream_t)stream));
  return FFMI_OK;
}

extern "C" ffmi_status ffmi_latent_attention(const void *q, const void *cache, int pages, void *o,
                                             int heads, int rank, float scale,
                                             const ffmi_paged_seq *seqs, int num_seqs,
                                             int full_precision) {
  using namespace ffmi;
  FFMI_CHECK(q && cache && o && seqs && num_seqs > 0 && heads > 0 && pages > 0 && rank > 0,
             FFMI_ERR_INVALID);
  FFMI_CHECK(rank % 32 == 0 && rank <= 2048, FFMI_ERR_UNSUPPORTED);
  const bool mfma = !full_precision && latent_rank_supported(rank);
  int T = 0, maxpos = 0;
  std::vector<PagedStep::Seg> segs;
  for (int i = 0; i < num_seqs; ++i) {
    FFMI_CHECK(seqs[i].num_tokens > 0 && seqs[i].pos0 >= 0 && seqs[i].pages, FFMI_ERR_INVALID);
    const int end = seqs[i].pos0 + seqs[i].num_tokens;
    for (int p = 0; p < (end + kPageTokens - 1) / kPageTokens; ++p)
      FFMI_CHECK(seqs[i].pages[p] >= 0 && seqs[i].pages[p] < pages, FFMI_ERR_INVALID);
    segs.push_back({seqs[i].num_tokens, seqs[i].pos0, seqs[i].pages});
    T += seqs[i].num_tokens;
    maxpos = std::max(maxpos, end);
  }
  constexpr int kSlots = 512;
  PagedStep step;
  ffmi_status st = step.init(T, num_seqs, maxpos, {RowShape{heads}}, mfma ? kSlots : 0);
  if (st != FFMI_OK) return st;
  std::vector<int32_t> ids(T, 0);
  st = step.stage(ids.data(), segs, nullptr, 0);
  if (st != FFMI_OK) return st;
  FFMI_HIP(hipMemcpy(step.dev, step.host, step.bytes, hipMemcpyHostToDevice));
  DeviceBuf slabs, ml;
  if (!slabs.get(mfma ? (size_t)kSlots * 64 * rank * 4 : 0) || !ml.get((size_t)kSlots * 64 * 8))
    return FFMI_ERR_OOM;
  if (mfma)
    FFMI_HIP(launch_latent_attention(step.dev, step.lists(heads), (const uint16_t *)q,
                                     (const uint16_t *)cache, (uint16_t *)o, (float *)slabs.p,
                                     (float *)ml.p, rank, scale, nullptr));
  else
    FFMI_HIP(launch_latent_attention_rows(step.dev, step.lists(heads), q, cache, o, rank, scale,
                                          !full_precision, nullptr));
  FFMI_HIP(hipDeviceSynchronize());
  return FFMI_OK;
}
