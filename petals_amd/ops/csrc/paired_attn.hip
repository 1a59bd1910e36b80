// Differential attention over paged keys and values: two softmax maps per head over the
// same values, a share of the second taken off the first, the result normed, scaled and
// gated (kernels: paged_attn.h).

#include "paged_attn.h"

// q [T, H, 2, dk]; the cache's keys [G, 2, dk]; out [T, >= H * dv] view, written up to H * dv:
// N(o_1 - share o_2) factor sigmoid(gate), N over a head's vdim values; gate [T, H] view in out's
// dtype, or none. Other arguments: paged_attention
void paired_attention(
    torch::Tensor q, torch::Tensor cache, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables,
    torch::Tensor tiles, int64_t run_tokens, int64_t max_keys, int64_t kv_heads, int64_t dv, int64_t chunk,
    double scale, double share, double factor, double eps, int64_t vdim, c10::optional<torch::Tensor> gate,
    torch::Tensor out, int64_t splits) {
  TORCH_CHECK(q.dim() == 4 && q.size(2) == 2 && chunk >= 0 && vdim >= 1 && vdim <= dv);
  AttnShape a = attn_shape(q.size(1), kv_heads, 2, q.size(3), dv, cache);
  a.chunk = chunk;
  a.scale = scale;
  a.share = share;
  a.factor = factor;
  a.eps = eps;
  a.vdim = vdim;
  run_attention<SOFTMAX, 2>(q, cache, pos, owner, tables, tiles, run_tokens, max_keys, a,
                            gated_out(out, gate, q.size(0), a), splits);
}
