// capi_fesenex.cpp -- C ABI of the gated bf16 product (include/ffmi.h): one
// operator at a time, for callers outside the models.
#include "../kernels/packing.h"
#include "device_buf.h"

extern "C" ffmi_status ffmi_linear_bf16_glu(const void *X, const void *W, void *Y, int T, int out_dim,
                                            int in_dim, float limit, ffmi_stream stream) {
  using namespace ffmi;
  FFMI_CHECK(X && W && Y && T > 0 && out_dim > 0 && in_dim > 0 && limit > 0.f, FFMI_ERR_INVALID);
  FFMI_CHECK(out_dim % 32 == 0 && in_dim % 32 == 0, FFMI_ERR_UNSUPPORTED);
  hipStream_t s = (hipStream_t)stream;
  const size_t wsb = gemm_bf16_glu_workspace_bytes(T, out_dim, in_dim);
  DeviceBuf xp, wp, ws;
  if (!xp.get((size_t)((T + 15) / 16) * 16 * in_dim * 2) || !wp.get((size_t)2 * out_dim * in_dim * 2) ||
      !ws.get(wsb))
    return FFMI_ERR_OOM;
  FFMI_HIP(launch_pack_act_bf16((const uint16_t *)X, (uint16_t *)xp.p, T, in_dim, s));
  PackSpec p;
  p.rows = p.cols = 1, p.nb = p.np = out_dim, p.kb = p.kp = in_dim;
  for (int k = 0; k < 2; ++k)
    FFMI_HIP(launch_pack_bf16((const uint16_t *)W + (size_t)k * out_dim * in_dim, in_dim, p,
                              (uint16_t *)wp.p, k, 2 * out_dim / 16, false, s, 2));
  FFMI_HIP(launch_gemm_bf16_glu((const uint16_t *)xp.p, (const uint16_t *)wp.p, (uint16_t *)Y, (float *)ws.p,
                                wsb, T, out_dim, in_dim, FFMI_X_PACKED, limit, s));
  FFMI_HIP(hipStreamSynchronize(s));  // (the packed operands are freed here)
  return FFMI_OK;
}
