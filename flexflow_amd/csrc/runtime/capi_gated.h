// capi_gated.h -- body of the C ABI's gated bf16 products: operands packed, one
// launch of `product` (X, W, ws), its end waited for.
#pragma once
#include "../kernels/packing.h"
#include "device_buf.h"

namespace ffmi {

template <class F>
ffmi_status gated_bf16_product(const void *X, const void *W, int T, int out_dim, int in_dim, size_t ws_bytes,
                               hipStream_t s, F product) {
  DeviceBuf xp, wp, ws;
  if (!xp.get((size_t)((T + 15) / 16) * 16 * in_dim * 2) || !wp.get((size_t)2 * out_dim * in_dim * 2) ||
      !ws.get(ws_bytes))
    return FFMI_ERR_OOM;
  FFMI_HIP(launch_pack_act_bf16((const uint16_t *)X, (uint16_t *)xp.p, T, in_dim, s));
  PackSpec p;
  p.rows = p.cols = 1, p.nb = p.np = out_dim, p.kb = p.kp = in_dim;
  for (int k = 0; k < 2; ++k)
    FFMI_HIP(launch_pack_bf16((const uint16_t *)W + (size_t)k * out_dim * in_dim, in_dim, p,
                              (uint16_t *)wp.p, k, 2 * out_dim / 16, false, s, 2));
  FFMI_HIP(product((const uint16_t *)xp.p, (const uint16_t *)wp.p, (float *)ws.p));
  FFMI_HIP(hipStreamSynchronize(s));  // (the packed operands are freed here)
  return FFMI_OK;
}

}  // namespace ffmi
