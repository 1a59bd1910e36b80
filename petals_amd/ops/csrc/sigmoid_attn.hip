// Attention over paged keys and values whose weights are sigmoids of the scores plus a
// bias per head, each for itself (kernels: paged_attn.h).

#include "paged_attn.h"

// bias [H] f32; out [T, >= H * dv] view, written up to H * dv; arguments: paged_attention
void sigmoid_attention(
    torch::Tensor q, torch::Tensor cache, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables,
    torch::Tensor tiles, int64_t run_tokens, int64_t max_keys, int64_t kv_heads, int64_t dv, int64_t chunk,
    double scale, torch::Tensor bias, torch::Tensor out, int64_t splits) {
  TORCH_CHECK(q.dim() == 3 && chunk >= 0);
  AttnShape a = attn_shape(q.size(1), kv_heads, 1, q.size(2), dv, cache);
  a.chunk = chunk;
  a.scale = scale;
  a.bias = opt_f32(bias, q.size(1));
  run_attention<SIGMOID, 1>(q, cache, pos, owner, tables, tiles, run_tokens, max_keys, a,
                            gated_out(out, c10::nullopt, q.size(0), a), splits);
}
