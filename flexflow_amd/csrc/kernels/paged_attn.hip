// paged_attn.hip -- attention with a bias by distance: launchers (kernels:
// paged_attn_kernels.h).
#include "paged_attn_kernels.h"

namespace ffmi {

hipError_t launch_attn_prep(const char *blob, int off_tokens, int T, const AttnPrep &a, bool f32,
                            hipStream_t s) {
  if (T <= 0) return hipSuccess;
  const int wide = std::max(std::max(a.dp, a.vp), std::max(a.dg, a.vg));
  if (wide > 1024 || a.y.S < 1 || a.y.S > 8 || a.every < 1) return hipErrorInvalidValue;
  const PagedToken *tok = reinterpret_cast<const PagedToken *>(blob + off_tokens);
#define FFMI_AP(E, NE, NT)                                                                           \
  hipLaunchKernelGGL((attn_prep_kernel<E, NE, NT>),                                                \
                     dim3((unsigned)(((long)((T + NT - 1) / NT) * (a.H + 2 * a.G) + 3) / 4)),      \
                     dim3(256), 0, s, tok, T, a)
#define FFMI_APN(E, NE)           \
  do {                            \
    if (T >= 128) FFMI_AP(E, NE, 4); \
    else FFMI_AP(E, NE, 1);       \
  } while (0)
  if (f32) {
    if (wide <= 256) FFMI_AP(float, 4, 1);
    else FFMI_AP(float, 16, 1);
  } else {
    if (wide <= 64) FFMI_APN(uint16_t, 1);
    else if (wide <= 128) FFMI_APN(uint16_t, 2);
    else if (wide <= 256) FFMI_APN(uint16_t, 4);
    else FFMI_AP(uint16_t, 16, 1);
  }
#undef FFMI_APN
#undef FFMI_AP
  return hipGetLastError();
}

hipError_t launch_paged_attn(const char *blob, const PagedLists &pl, const AttnArgs &a, float *slabs,
                             float *ml, hipStream_t s, const AttnPrep *pr, int T) {
  return launch_attn_kind<kBias>(blob, pl, a, slabs, ml, s, pr, T);
}
hipError_t launch_paged_attn_rows(const char *blob, const PagedLists &pl, const AttnArgs &a, bool f32,
                                  hipStream_t s) {
  return launch_attn_rows_kind<kBias>(blob, pl, a, f32, s);
}

}  // namespace ffmi
