// conv_rows.hip -- causal convolution over time of a product's columns (conv_rows.h).
#include "conv_rows.h"

#include "device_util.h"

namespace ffmi {

// A thread has 8 columns of TB tokens.  PAST: taps - 1, the earlier rows and the weights in
// registers; or -1: read again.
template <int PAST, bool F32>
__global__ __launch_bounds__(256) void conv_rows_kernel(const char *__restrict__ blob, ConvRows a) {
  constexpr int TB = 8, H = PAST > 0 ? PAST : 1;
  const int c = (blockIdx.x * 256 + threadIdx.x) * 8, t0 = blockIdx.y * TB;
  if (c >= a.cols) return;
  const PagedToken *tok = reinterpret_cast<const PagedToken *>(blob + a.off_tokens);
  const size_t slab = (size_t)a.T * a.u.NP;
  const int past = a.taps - 1;
  auto load8 = [](const float *p, f4 (&v)[2]) {
    v[0] = *reinterpret_cast<const f4 *>(p), v[1] = *reinterpret_cast<const f4 *>(p + 4);
  };
  auto row = [&](int t, f4 (&v)[2]) {
    const float *p = a.u.p + (size_t)t * a.u.NP + a.col + c;
    load8(p, v);
    for (int s = 1; s < a.u.S; ++s) {
      f4 w[2];
      load8(p + s * slab, w);
      v[0] += w[0], v[1] += w[1];
    }
  };
  // the row d tokens before token t
  auto before = [&](const PagedToken &tk, int t, int d, f4 (&v)[2]) {
    v[0] = v[1] = f4{0.f, 0.f, 0.f, 0.f};
    if (tk.back >= d) row(t - d, v);
    else if (tk.pos >= d) load8(a.carry + (((size_t)tk.slot * 2 + tk.bank) * past + d - tk.back - 1) * a.cols + c, v);
  };
  f4 u[TB][2], x[H][2], wt[H + 1][2];
#pragma unroll
  for (int k = 0; k < TB; ++k) row(min(t0 + k, a.T - 1), u[k]);
  if constexpr (PAST >= 0)
#pragma unroll
    for (int d = 0; d <= PAST; ++d) load8(a.conv + (size_t)(PAST - d) * a.cols + c, wt[d]);
#pragma unroll
  for (int k = 0; k < TB; ++k) {
    const int t = t0 + k;
    if (t >= a.T) break;
    const PagedToken tk = tok[t];
    if (PAST > 0 && (k == 0 || tk.back == 0))
#pragma unroll
      for (int d = 1; d <= PAST; ++d) before(tk, t, d, x[d - 1]);
    if (tk.back + tk.ahead + 1 > a.above) {
      float *now = a.carry + ((size_t)tk.slot * 2 + (tk.bank ^ 1)) * past * a.cols + c;
      auto keep = [&](int place, const f4 (&v)[2]) {
        float *p = now + (size_t)place * a.cols;
        *reinterpret_cast<f4 *>(p) = v[0], *reinterpret_cast<f4 *>(p + 4) = v[1];
      };
      f4 v[2], e[2];
      if (tk.ahead < past) keep(tk.ahead, u[k]);
      if constexpr (PAST >= 0) {
        if (tk.back == 0)  // (a short portion: earlier rows move on)
#pragma unroll
          for (int d = 1; d <= PAST; ++d)
            if (tk.ahead + d < PAST) keep(tk.ahead + d, x[d - 1]);
        v[0] = u[k][0] * wt[0][0], v[1] = u[k][1] * wt[0][1];
#pragma unroll
        for (int d = 1; d <= PAST; ++d) v[0] += x[d - 1][0] * wt[d][0], v[1] += x[d - 1][1] * wt[d][1];
      } else {
        load8(a.conv + (size_t)past * a.cols + c, e);
        v[0] = u[k][0] * e[0], v[1] = u[k][1] * e[1];
        for (int d = 1; d <= past; ++d) {
          f4 w[2];
          before(tk, t, d, e);
          if (tk.back == 0 && tk.ahead + d < past) keep(tk.ahead + d, e);
          load8(a.conv + (size_t)(past - d) * a.cols + c, w);
          v[0] += e[0] * w[0], v[1] += e[1] * w[1];
        }
      }
      if (a.silu)
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const float z = v[i >> 2][i & 3];
          if constexpr (F32) v[i >> 2][i & 3] = silu_f(z);
          else v[i >> 2][i & 3] = z * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.44269504f * z));
        }
      if constexpr (F32) {
        float *p = a.hf + (size_t)t * a.cols + c;
        *reinterpret_cast<f4 *>(p) = v[0], *reinterpret_cast<f4 *>(p + 4) = v[1];
      } else {
        *reinterpret_cast<uint4 *>(a.hb + (size_t)t * a.cols + c) = pack8_bf16(v[0], v[1]);
      }
    }
    if constexpr (PAST > 0) {
#pragma unroll
      for (int d = PAST; d > 1; --d) x[d - 1][0] = x[d - 2][0], x[d - 1][1] = x[d - 2][1];
      x[0][0] = u[k][0], x[0][1] = u[k][1];
    }
  }
}

hipError_t launch_conv_rows(const char *blob, const ConvRows &a, hipStream_t s) {
  if (a.T <= 0) return hipSuccess;
  if (a.cols <= 0 || a.cols % 8 || a.col % 4 || a.u.NP % 4 || a.u.S < 1 || a.col + a.cols > a.u.NP || a.taps < 1 ||
      !a.conv || (a.taps > 1 && !a.carry) || (a.hb != nullptr) == (a.hf != nullptr))
    return hipErrorInvalidValue;
  const dim3 grid((a.cols + 2047) / 2048, (a.T + 7) / 8);
#define FFMI_CR(PAST)                                                                           \
  do {                                                                                          \
    if (a.hf) hipLaunchKernelGGL((conv_rows_kernel<PAST, true>), grid, dim3(256), 0, s, blob, a); \
    else hipLaunchKernelGGL((conv_rows_kernel<PAST, false>), grid, dim3(256), 0, s, blob, a);   \
  } while (0)
  if (a.taps == 1) FFMI_CR(0);
  else if (a.taps == 2) FFMI_CR(1);
  else if (a.taps == 3) FFMI_CR(2);
  else if (a.taps == 4) FFMI_CR(3);
  else FFMI_CR(-1);
#undef FFMI_CR
  return hipGetLastError();
}

}  // namespace ffmi
