#include "paged_attn.inc"

int launch_diff_attn_f32(const PagedAttnArgs& a, hipStream_t stream) {
  return launch_dims<float, 2>(a, stream);
}
