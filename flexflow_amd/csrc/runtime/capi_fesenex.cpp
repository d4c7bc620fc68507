// capi_fesenex.cpp -- C ABI of the gated bf16 product (include/ffmi.h): one
// operator at a time, for callers outside the models.
#include "capi_gated.h"

extern "C" ffmi_status ffmi_linear_bf16_glu(const void *X, const void *W, void *Y, int T, int out_dim,
                                            int in_dim, float limit, ffmi_stream stream) {
  using namespace ffmi;
  FFMI_CHECK(X && W && Y && T > 0 && out_dim > 0 && in_dim > 0 && limit > 0.f, FFMI_ERR_INVALID);
  FFMI_CHECK(out_dim % 32 == 0 && in_dim % 32 == 0, FFMI_ERR_UNSUPPORTED);
  hipStream_t s = (hipStream_t)stream;
  const size_t wsb = gemm_bf16_glu_workspace_bytes(T, out_dim, in_dim);
  return gated_bf16_product(X, W, T, out_dim, in_dim, wsb, s, [&](const uint16_t *x, const uint16_t *w, float *ws) {
    return launch_gemm_bf16_glu(x, w, (uint16_t *)Y, ws, wsb, T, out_dim, in_dim, FFMI_X_PACKED, limit, s);
  });
}
