#include "paged_attn.inc"

int launch_slope_attn_bf16(const PagedAttnArgs& a, hipStream_t stream) {
  return launch_dims<bf16, 1, true>(a, stream);
}
