// Rows of latent attention whose queries pass through a latent of their own and
// whose keys have a rotated part that all heads share (CDNA4, gfx950).
//
//   latent_rows     per token: the query latent, normed; the key/value latent, normed,
//                   and the rotated key part into their page; the heads' output gates
//   rotate_queries  the rotated part of the queries behind their latent part
//
// Rotation: rotary.h.

#include "common.h"
#include "paged.h"
#include "rotary.h"
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>

// value d of a row of rotated values
template <typename T>
__device__ __forceinline__ float rotated(const T* x, int d, int pos, const Rotation& r) {
  const int half = r.turned / 2;
  if (d >= 2 * half) return load_f32(x + d);
  const int i = d < half ? d : d - half;
  float s, c;
  sin_cos(pos * r.quarters[i], s, c);
  const float u = load_f32(x + i), v = load_f32(x + i + half);
  return d < half ? u * c - v * s : fmaf(v, c, u * s);
}

struct LatentColumns {
  int q, q_rank, q_pad;    // query latent: first column, size, size of its padded rows
  int kv, kv_rank, kv_pad; // key/value latent, then the rotated part; kv < 0: none
  int rot;                 // values of the rotated part
  int gate, heads;
};

// One workgroup of NT threads per token.
template <typename TY, typename TC, typename TQ, int NT>
__global__ __launch_bounds__(NT) void latent_rows_kernel(
    const TY* __restrict__ y, int stride, LatentColumns n, const float* __restrict__ w_q, const float* __restrict__ w_kv,
    Rotation rot, TC* __restrict__ cache, int width, PagedRows b, TQ* __restrict__ cq, float* __restrict__ factor,
    float eps) {
  __shared__ float red[2][NT / WAVE];
  const int tid = threadIdx.x;
  const size_t t = blockIdx.x;
  const TY* row = y + t * stride;
  float q2 = 0.f, c2 = 0.f;
  for (int d = tid; d < n.q_rank; d += NT) {
    const float v = load_f32(row + n.q + d);
    q2 = fmaf(v, v, q2);
  }
  if (n.kv >= 0)
    for (int d = tid; d < n.kv_rank; d += NT) {
      const float v = load_f32(row + n.kv + d);
      c2 = fmaf(v, v, c2);
    }
  q2 = wave_reduce_sum(q2);
  c2 = wave_reduce_sum(c2);
  if ((tid & (WAVE - 1)) == 0) {
    red[0][tid / WAVE] = q2;
    red[1][tid / WAVE] = c2;
  }
  __syncthreads();
  q2 = c2 = 0.f;
#pragma unroll
  for (int i = 0; i < NT / WAVE; ++i) {
    q2 += red[0][i];
    c2 += red[1][i];
  }
  const float iq = 1.f / sqrtf(q2 / n.q_rank + eps);
  for (int d = tid; d < n.q_pad; d += NT)
    store_f32(cq + t * n.q_pad + d, d < n.q_rank ? load_f32(row + n.q + d) * iq * w_q[d] : 0.f);
  for (int h = tid; h < n.heads; h += NT) factor[t * n.heads + h] = 1.f / (1.f + expf(-load_f32(row + n.gate + h)));
  if (n.kv < 0) return;
  const int pos = b.pos[t];
  const long at = cache_row(b, b.owner[t], pos);
  if (at < 0) return;
  const float ic = 1.f / sqrtf(c2 / n.kv_rank + eps);
  TC* dst = cache + (size_t)at * width;
  for (int d = tid; d < n.kv_pad; d += NT)
    store_f32(dst + d, d < n.kv_rank ? load_f32(row + n.kv + d) * ic * w_kv[d] : 0.f);
  for (int d = tid; d < width - n.kv_pad; d += NT)
    store_f32(dst + n.kv_pad + d, d < n.rot ? rotated(row + n.kv + n.kv_rank, d, pos, rot) : 0.f);
}

// One workgroup per token; a thread turns one pair of every (256 / columns)th head,
// where a row's columns are its pairs and, behind them, the values that pass.
template <typename TY, typename TQ>
__global__ __launch_bounds__(256) void rotate_queries_kernel(
    const TY* __restrict__ y, int stride, int first, int heads, int rot_pad, Rotation rot, const int* __restrict__ pos,
    TQ* __restrict__ q, int width, int offset) {
  const size_t t = blockIdx.x;
  const int half = rot.turned / 2, columns = rot_pad - half, p = pos[t];
  const int per = max(1, 256 / columns), h0 = threadIdx.x / columns;
  if (columns <= 256 && h0 >= per) return;
  const TY* src = y + t * stride + first;
  TQ* dst = q + t * heads * width + offset;
  for (int i = columns <= 256 ? threadIdx.x - h0 * columns : threadIdx.x; i < columns; i += 256) {
    const bool pair = i < half;
    float s = 0.f, c = 1.f;
    if (pair) sin_cos(p * rot.quarters[i], s, c);
#pragma unroll 4
    for (int h = columns <= 256 ? h0 : 0; h < heads; h += per) {
      const TY* x = src + h * rot_pad;
      TQ* o = dst + (size_t)h * width;
      if (pair) {
        const float u = load_f32(x + i), v = load_f32(x + i + half);
        store_f32(o + i, u * c - v * s);
        store_f32(o + i + half, fmaf(v, c, u * s));
      } else {
        store_f32(o + i + half, load_f32(x + i + half));
      }
    }
  }
}

// ------------------------------------------------------------------- host

static bool f32_rows(const torch::Tensor& t) {
  TORCH_CHECK(t.is_cuda() && (t.dtype() == torch::kFloat32 || t.dtype() == torch::kBFloat16));
  return t.dtype() == torch::kFloat32;
}

// y [T, n]: the projections; at_q, at_kv (-1: none), at_gate: first columns in it.
// Returns (query latent [T, q_pad], gates [T, heads] 32-bit).
std::vector<torch::Tensor> latent_rows(
    torch::Tensor y, int64_t at_q, torch::Tensor w_q, int64_t q_pad, bool q_f32, int64_t at_kv,
    c10::optional<torch::Tensor> w_kv, int64_t kv_pad, int64_t rot, torch::Tensor quarters, torch::Tensor cache,
    int64_t at_gate, int64_t heads, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables, double eps) {
  const bool yf = f32_rows(y), cf = f32_rows(cache);
  TORCH_CHECK(y.dim() == 2 && y.is_contiguous());
  const long t = y.size(0), width = y.size(1);
  const PagedRows b = paged_rows(pos, owner, tables, cache, t);
  LatentColumns n;
  n.q = at_q, n.q_rank = w_q.numel(), n.q_pad = q_pad;
  n.kv = at_kv, n.kv_rank = 1, n.kv_pad = kv_pad, n.rot = rot, n.gate = at_gate, n.heads = heads;
  TORCH_CHECK(w_q.is_cuda() && w_q.dtype() == torch::kFloat32 && w_q.is_contiguous());
  TORCH_CHECK(at_q >= 0 && at_q + n.q_rank <= width && n.q_rank >= 1 && q_pad >= n.q_rank);
  TORCH_CHECK(at_gate >= 0 && at_gate + heads <= width);
  const float* wkv = nullptr;
  const Rotation r = rotation(quarters);
  if (at_kv >= 0) {
    TORCH_CHECK(w_kv.has_value() && w_kv->is_cuda() && w_kv->dtype() == torch::kFloat32 && w_kv->is_contiguous());
    n.kv_rank = w_kv->numel();
    wkv = w_kv->data_ptr<float>();
    TORCH_CHECK(n.kv_rank >= 1 && at_kv + n.kv_rank + rot <= width && kv_pad >= n.kv_rank && kv_pad + rot <= cache.size(2));
    TORCH_CHECK(r.turned <= rot, "rotation of ", r.turned, " of ", rot, " values");
  }
  auto cq = torch::empty({t, q_pad}, y.options().dtype(q_f32 ? torch::kFloat32 : torch::kBFloat16));
  auto factor = torch::empty({t, heads}, y.options().dtype(torch::kFloat32));
  if (t == 0) return {cq, factor};
  auto stream = at::cuda::getCurrentCUDAStream();
#define LRN(TY, TC, TQ, NT)                                                                                  \
  latent_rows_kernel<TY, TC, TQ, NT><<<t, NT, 0, stream>>>(                                                  \
      reinterpret_cast<const TY*>(y.data_ptr()), (int)width, n, w_q.data_ptr<float>(), wkv, r,               \
      reinterpret_cast<TC*>(cache.data_ptr()), (int)cache.size(2), b, reinterpret_cast<TQ*>(cq.data_ptr()),  \
      factor.data_ptr<float>(), (float)eps)
#define LR(TY, TC, TQ)                    \
  do {                                    \
    if (t < 512) LRN(TY, TC, TQ, 1024);   \
    else LRN(TY, TC, TQ, 256);            \
  } while (0)
#define LRQ(TY, TC)                       \
  do {                                    \
    if (q_f32) LR(TY, TC, float);         \
    else LR(TY, TC, unsigned short);      \
  } while (0)
  if (yf && cf) LRQ(float, float);
  else if (yf) LRQ(float, unsigned short);
  else if (cf) LRQ(unsigned short, float);
  else LRQ(unsigned short, unsigned short);
#undef LRQ
#undef LR
#undef LRN
  HIP_CHECK_LAST();
  return {cq, factor};
}

// columns [first, first + heads * rot_pad) of y, head by head, rotated into
// q[:, :, offset : offset + rot_pad]
void rotate_queries(torch::Tensor y, int64_t first, int64_t rot_pad, torch::Tensor quarters, torch::Tensor pos,
                    torch::Tensor q, int64_t offset) {
  const bool yf = f32_rows(y), qf = f32_rows(q);
  TORCH_CHECK(y.dim() == 2 && y.is_contiguous() && q.dim() == 3 && q.is_contiguous() && y.size(0) == q.size(0));
  const long t = q.size(0), heads = q.size(1);
  TORCH_CHECK(first >= 0 && first + heads * rot_pad <= y.size(1) && offset >= 0 && offset + rot_pad <= q.size(2));
  TORCH_CHECK(pos.is_cuda() && pos.dtype() == torch::kInt32 && pos.is_contiguous() && pos.numel() == t);
  const Rotation r = rotation(quarters);
  TORCH_CHECK(r.turned <= rot_pad, "rotation of ", r.turned, " of ", rot_pad, " values");
  if (t == 0 || rot_pad == 0) return;
  auto stream = at::cuda::getCurrentCUDAStream();
#define RQ(TY, TQ)                                                                                                \
  rotate_queries_kernel<TY, TQ><<<t, 256, 0, stream>>>(                                                           \
      reinterpret_cast<const TY*>(y.data_ptr()), (int)y.size(1), (int)first, (int)heads, (int)rot_pad, r,         \
      pos.data_ptr<int>(), reinterpret_cast<TQ*>(q.data_ptr()), (int)q.size(2), (int)offset)
  if (yf && qf) RQ(float, float);
  else if (yf) RQ(float, unsigned short);
  else if (qf) RQ(unsigned short, float);
  else RQ(unsigned short, unsigned short);
#undef RQ
  HIP_CHECK_LAST();
}
