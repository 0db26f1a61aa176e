#include "paged_attn.inc"

int launch_diff_attn_bf16(const PagedAttnArgs& a, hipStream_t stream) {
  return launch_dims<bf16, 2>(a, stream);
}
