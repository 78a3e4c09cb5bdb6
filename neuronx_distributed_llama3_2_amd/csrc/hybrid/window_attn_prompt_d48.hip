// Prompt attention for query / key sizes up to 48 (window_attn_prompt.h).
#include "window_attn_prompt.h"

namespace nxd {
int attn_prompt_d48_launch(const WindowAttnParams& p, hipStream_t s) {
  if (p.pool > 0) return hybrid::attn_prompt_pooled<3>(p, s);
  if (p.maps == 1) return hybrid::attn_prompt_by_v<3, 1, false>(p, s);
  return p.softcap > 0.f && p.softcap <= 40.f ? hybrid::attn_prompt_by_v<3, 2, true>(p, s)
                                              : hybrid::attn_prompt_by_v<3, 2, false>(p, s);
}
}  // namespace nxd
