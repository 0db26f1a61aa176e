#include "paged_attn.inc"

int launch_slope_attn_f32(const PagedAttnArgs& a, hipStream_t stream) {
  return launch_dims<float, 1, true>(a, stream);
}
