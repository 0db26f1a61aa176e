#include "row_attn.inc"

int launch_latent_attn_f32(const RowAttnArgs& a, hipStream_t stream) {
  return launch_latent_dims<float>(a, stream);
}

int launch_head_attn_f32(const RowAttnArgs& a, hipStream_t stream) {
  return launch_heads_dims<float>(a, stream);
}
