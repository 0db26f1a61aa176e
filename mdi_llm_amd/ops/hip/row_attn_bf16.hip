#include "row_attn.inc"

int launch_latent_attn_bf16(const RowAttnArgs& a, hipStream_t stream) {
  return launch_latent_dims<bf16>(a, stream);
}

int launch_head_attn_bf16(const RowAttnArgs& a, hipStream_t stream) {
  return launch_heads_dims<bf16>(a, stream);
}
