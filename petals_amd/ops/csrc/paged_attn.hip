// Softmax attention over paged keys and values with a sliding window, a bias per head
// that grows with the distance, a sink and a gate (kernels: paged_attn.h), and the rows
// that it reads:
//
//   attn_prepare        bias, query temperature, value mixing; writes the cache

#include "paged_attn.h"
#include <ATen/cuda/CUDAContext.h>

// ------------------------------------------------------- queries and cache

struct MixValues {
  const float* lambda;  // null: values are not mixed
  float* first;         // a row's first-layer values: first[t * stride + kvh * vdim + c], or null
  long stride;
  int vdim;             // unpadded
  bool aligned;         // groups of 8 of `first` may be moved at once
};

// y [T, >= H*dk + G*(dk+dv)]: queries, keys, values. 8 columns per thread; a
// group of 8 lies in one head. lambda null and first given: values are stored there.
template <typename TY, typename TC>
__global__ __launch_bounds__(256) void attn_prepare_kernel(
    const TY* __restrict__ y, int y_stride, const float* __restrict__ bias, TC* __restrict__ q,
    TC* __restrict__ cache, PagedRows b, AttnShape a, MixValues mix, float temp_coef, int temp_every) {
  const int nq = a.heads * a.dk, nk = a.kv_heads * a.dk, nv = a.kv_heads * a.dv;
  const int c0 = (blockIdx.x * 256 + threadIdx.x) * 8;
  if (c0 >= nq + nk + nv) return;
  const size_t t = blockIdx.y;
  const int pos = b.pos[t];
  float v[8], w[8];
  load8(y + t * y_stride + c0, v);
  load8(bias + c0, w);
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] += w[e];
  TC* dst;
  if (c0 < nq) {
    if (temp_coef != 0.f) {
      const float f = 1.f + temp_coef * logf((float)((pos + 1) / temp_every) + 1.f);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] *= f;
    }
    dst = q + t * nq + c0;
  } else {
    const long row = cache_row(b, b.owner[t], pos);
    const int c = c0 - nq - nk;  // column among the values
    if (c >= 0 && mix.first) {
      const int kvh = c / a.dv, d0 = c - kvh * a.dv;
      float* own = mix.first + t * mix.stride + kvh * mix.vdim + d0;
      const float lam = mix.lambda ? *mix.lambda : 0.f;
      if (mix.aligned && d0 + 8 <= mix.vdim) {
        if (mix.lambda) {
          load8(own, w);
#pragma unroll
          for (int e = 0; e < 8; ++e) v[e] = (1.f - lam) * v[e] + lam * w[e];
        } else {
          store8(own, v);
        }
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e)
          if (d0 + e < mix.vdim) {
            if (mix.lambda) v[e] = (1.f - lam) * v[e] + lam * own[e];
            else own[e] = v[e];
          }
      }
    }
    if (row < 0) return;
    dst = cache + (size_t)row * (nk + nv) + (c0 - nq);
  }
  store8(dst, v);
}

// ------------------------------------------------------------------- host

torch::Tensor paged_attention(
    torch::Tensor q,       // [T, H, dk] bf16 or f32
    torch::Tensor cache,   // [pages, PAGE, G * (dk + dv)], dtype of q
    torch::Tensor pos, torch::Tensor owner, torch::Tensor tables,
    torch::Tensor tiles,   // [n, 2] int32 runs of at most run_tokens tokens
    int64_t run_tokens,
    int64_t max_keys,      // most keys that any row sees
    int64_t kv_heads, int64_t dv, int64_t window, double scale,
    c10::optional<torch::Tensor> slopes, c10::optional<torch::Tensor> sink,
    c10::optional<torch::Tensor> gate,  // [T, H * dv] view, unit column stride; the result has its dtype
    bool out_f32, int64_t splits) {
  TORCH_CHECK(q.dim() == 3);
  const long t = q.size(0), heads = q.size(1);
  AttnShape a = attn_shape(heads, kv_heads, 1, q.size(2), dv, cache);
  a.window = window;
  a.scale = scale;
  a.slopes = opt_f32(slopes, heads);
  a.sink = opt_f32(sink, heads);
  auto out = torch::empty({t, heads * dv}, q.options().dtype(out_f32 ? torch::kFloat32 : torch::kBFloat16));
  run_attention<SOFTMAX, 1>(q, cache, pos, owner, tables, tiles, run_tokens, max_keys, a, gated_out(out, gate, t, a),
                            splits);
  return out;
}

// Returns the queries [T, H, dk] in the cache's dtype; keys and values go to the cache.
torch::Tensor attn_prepare(
    torch::Tensor y,       // [T, ys] f32 or bf16; columns: H*dk queries, G*dk keys, G*dv values
    torch::Tensor bias,    // [>= those columns] f32
    torch::Tensor cache, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables,
    int64_t heads, int64_t kv_heads, int64_t dk, int64_t dv, double temp_coef, int64_t temp_every,
    c10::optional<torch::Tensor> first,   // [T, >= G*vdim] f32 view with unit column stride
    c10::optional<torch::Tensor> lambda,  // one f32 value; absent: `first` is written
    int64_t vdim) {
  const bool yf = f32_or_bf16(y), cf = f32_or_bf16(cache);
  const int t = y.size(0);
  TORCH_CHECK(y.dim() == 2 && y.is_contiguous() && temp_every >= 1);
  const PagedRows b = paged_rows(pos, owner, tables, cache, t);
  const AttnShape a = attn_shape(heads, kv_heads, 1, dk, dv, cache);
  const long cols = heads * dk + kv_heads * (dk + dv);
  TORCH_CHECK(y.size(1) >= cols && y.size(1) % 8 == 0, "projection too narrow");
  for (const auto& p : {y, bias, cache}) TORCH_CHECK(reinterpret_cast<uintptr_t>(p.data_ptr()) % 16 == 0);
  TORCH_CHECK(bias.is_cuda() && bias.dtype() == torch::kFloat32 && bias.is_contiguous() && bias.numel() >= cols);
  MixValues mix{nullptr, nullptr, 0, (int)vdim, false};
  if (first.has_value()) {
    TORCH_CHECK(first->is_cuda() && first->dtype() == torch::kFloat32 && first->dim() == 2 && first->stride(1) == 1);
    TORCH_CHECK(first->size(0) == t && first->size(1) >= kv_heads * vdim && vdim <= dv);
    mix.first = first->data_ptr<float>();
    mix.stride = first->stride(0);
    mix.aligned = vdim % 8 == 0 && mix.stride % 4 == 0 && reinterpret_cast<uintptr_t>(mix.first) % 16 == 0;
    if (lambda.has_value()) {
      TORCH_CHECK(lambda->is_cuda() && lambda->dtype() == torch::kFloat32 && lambda->numel() == 1);
      mix.lambda = lambda->data_ptr<float>();
    }
  }
  auto q = torch::empty({t, (long)heads, (long)dk}, cache.options());
  TORCH_CHECK(t <= 65535, "at most 65535 rows in a step");
  if (t == 0) return q;
  const dim3 grid((cols / 8 + 255) / 256, t);
  auto stream = at::cuda::getCurrentCUDAStream();
#define AP(TY, TC, YP, QP, CP)                                                                                \
  attn_prepare_kernel<TY, TC><<<grid, 256, 0, stream>>>(YP, (int)y.size(1), bias.data_ptr<float>(), QP, CP, b, a, mix, \
                                                        (float)temp_coef, (int)temp_every)
  if (yf && cf) AP(float, float, y.data_ptr<float>(), q.data_ptr<float>(), cache.data_ptr<float>());
  else if (yf) AP(float, unsigned short, y.data_ptr<float>(), BF16P(q), BF16P(cache));
  else if (cf) AP(unsigned short, float, BF16P(y), q.data_ptr<float>(), cache.data_ptr<float>());
  else AP(unsigned short, unsigned short, BF16P(y), BF16P(q), BF16P(cache));
#undef AP
  HIP_CHECK_LAST();
  return q;
}
