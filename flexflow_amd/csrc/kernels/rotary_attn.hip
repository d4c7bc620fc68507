// rotary_attn.hip -- attention with rotated queries and keys: launchers (kernels:
// paged_attn_kernels.h).
#include "paged_attn_kernels.h"

namespace ffmi {

hipError_t launch_rotary_prep(const char *blob, int off_tokens, int T, const AttnPrep &a, bool f32,
                              hipStream_t s) {
  if (T <= 0) return hipSuccess;
  const int wide = std::max(std::max(a.dp, a.vp), std::max(a.dg, a.vg));
  if (wide > 1024 || a.y.S < 1 || a.y.S > 8 || a.rot < 0 || a.rot > a.dim || a.rot % 2 || (a.rot && !a.freq) ||
      a.taps > 0)
    return hipErrorInvalidValue;
  const PagedToken *tok = reinterpret_cast<const PagedToken *>(blob + off_tokens);
  const int runs = (a.H + 2 * a.G + 7) / 8;  // of eight heads
#define FFMI_RP(E, NE, NT)                                                                        \
  do {                                                                                            \
    const int nt = (T + NT - 1) / NT;                                                             \
    const int gy = std::min(runs, std::max(1, 512 / nt)); /* fill the chip */                     \
    hipLaunchKernelGGL((rotary_prep_kernel<E, NE, NT>), dim3(nt, gy), dim3(512), 0, s, tok, T, a); \
  } while (0)
#define FFMI_RPN(E, NE)              \
  do {                               \
    if (T >= 128) FFMI_RP(E, NE, 4); \
    else FFMI_RP(E, NE, 1);          \
  } while (0)
  if (f32) {
    if (wide <= 256) FFMI_RP(float, 4, 1);
    else FFMI_RP(float, 16, 1);
  } else {
    if (wide <= 64) FFMI_RPN(uint16_t, 1);
    else if (wide <= 128) FFMI_RPN(uint16_t, 2);
    else if (wide <= 256) FFMI_RPN(uint16_t, 4);
    else FFMI_RP(uint16_t, 16, 1);
  }
#undef FFMI_RPN
#undef FFMI_RP
  return hipGetLastError();
}

hipError_t launch_rotary_attn(const char *blob, const PagedLists &pl, const AttnArgs &a, float *slabs,
                              float *ml, hipStream_t s, const AttnPrep *pr, int T) {
  return launch_attn_kind<kRotary>(blob, pl, a, slabs, ml, s, pr, T);
}
hipError_t launch_rotary_attn_rows(const char *blob, const PagedLists &pl, const AttnArgs &a, bool f32,
                                   hipStream_t s) {
  return launch_attn_rows_kind<kRotary>(blob, pl, a, f32, s);
}

}  // namespace ffmi
