// Prompt-row attention with fp32 operands for key and value heads of different sizes (attn_rows.h): the smallest
// compiled pair of sizes (32, 64, 128, 256) that holds both.
#include "attn_rows.h"

namespace cthip {

template <int DK, int DV>
static void go(const AttnRowsArgs &a) {
  constexpr int NW = DK <= 64 && DV <= 64 ? 8 : 4;  // wavefronts whose key tiles fit LDS together
  hipLaunchKernelGGL((k_attn_mfma<DK, DV, NW, true>), dim3(a.H, (a.S + 31) / 32), dim3(64 * NW), 0, state().stream, a);
}
template <int DK>
static void go_k(const AttnRowsArgs &a) {
  if (a.dv <= 32) go<DK, 32>(a);
  else if (a.dv <= 64) go<DK, 64>(a);
  else if (a.dv <= 128) go<DK, 128>(a);
  else go<DK, 256>(a);
}
int launch_attn_rows_f32(const AttnRowsArgs &a) {
  if (a.dk <= 32) go_k<32>(a);
  else if (a.dk <= 64) go_k<64>(a);
  else if (a.dk <= 128) go_k<128>(a);
  else go_k<256>(a);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

int launch_attn_rows(const AttnRowsArgs &a, bool fp32_operands) {
  if (a.S <= 0) return 0;
  if (a.dk > 256 || a.dv > 256 || (a.dk & 3) || (a.dv & 3)) return fail(CTHIP_E_UNSUPPORTED, "attention: key / value heads of %d / %d (multiples of 4 up to 256)", a.dk, a.dv);
  return fp32_operands ? launch_attn_rows_f32(a) : launch_attn_rows_bf(a);
}

}  // namespace cthip
