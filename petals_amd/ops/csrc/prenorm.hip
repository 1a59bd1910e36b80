// Sublayer kernels for blocks that norm each sublayer's INPUT and keep the
// residual stream in 32-bit (CDNA4, gfx950).
//
//   residual_norm   x += mult (y + bias), y one matrix or several to be summed, then RMS
//                   norm of x with a plain weight, of the whole row or of equal parts of it
//   residual_sum    x += mult (split-K partial sums + bias) of a decoding product
//   bias_relu2      relu(y + bias)^2
//   bias_xielu      xIELU of y + bias, y a matrix (in place) or split-K partial sums
//
// The stream's rows may be wider than the residual (what lies past it is left
// alone); the norm is written in rows padded with zeros to a multiple of 8.

#include "common.h"
#include "paged.h"
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>

__device__ __forceinline__ f32x4 load4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ f32x4 load4(const unsigned short* p) {
  const v4s a = *reinterpret_cast<const v4s*>(p);
  return f32x4{bf16_to_f32(a[0]), bf16_to_f32(a[1]), bf16_to_f32(a[2]), bf16_to_f32(a[3])};
}
__device__ __forceinline__ void store4(float* p, f32x4 v) { *reinterpret_cast<f32x4*>(p) = v; }
__device__ __forceinline__ void store4(unsigned short* p, f32x4 v) {
  *reinterpret_cast<v4s*>(p) = v4s{(short)f32_to_bf16(v[0]), (short)f32_to_bf16(v[1]), (short)f32_to_bf16(v[2]),
                                   (short)f32_to_bf16(v[3])};
}

// One workgroup per token. y null: x is only read; h null: nothing is normed. y: `parts`
// matrices, part_stride apart.
template <typename TY, typename TH>
__global__ __launch_bounds__(1024) void residual_norm_kernel(
    float* __restrict__ x, long x_stride, const TY* __restrict__ y, long y_stride, const float* __restrict__ bias,
    const float* __restrict__ w, float eps, TH* __restrict__ h, int d, int dp, bool by4, float mult, int groups,
    int parts, long part_stride) {
  extern __shared__ float row[];  // [d], then of each group
  __shared__ float red[16];
  const int tid = threadIdx.x, nt = blockDim.x;
  const size_t t = blockIdx.x;
  float* xr = x + t * x_stride;
  float ss = 0.f;
  if (by4) {
    for (int c = tid * 4; c < d; c += nt * 4) {
      f32x4 v = load4(xr + c);
      if (y) {
        f32x4 u = load4(y + t * y_stride + c);
        const f32x4 b = bias ? load4(bias + c) : f32x4{0.f, 0.f, 0.f, 0.f};
        for (int i = 1; i < parts; ++i) {
          const f32x4 more = load4(y + i * part_stride + t * y_stride + c);
#pragma unroll
          for (int e = 0; e < 4; ++e) u[e] += more[e];
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = fmaf(mult, u[e] + b[e], v[e]);
        store4(xr + c, v);
      }
      store4(row + c, v);
#pragma unroll
      for (int e = 0; e < 4; ++e) ss = fmaf(v[e], v[e], ss);
    }
  }
  for (int c = by4 ? d : tid; c < d; c += nt) {
    float v = xr[c];
    if (y) {
      float u = load_f32(y + t * y_stride + c);
      for (int i = 1; i < parts; ++i) u += load_f32(y + i * part_stride + t * y_stride + c);
      v = fmaf(mult, u + (bias ? bias[c] : 0.f), v);
      xr[c] = v;
    }
    row[c] = v;
    ss = fmaf(v, v, ss);
  }
  if (!h) return;  // uniform
  if (groups > 1) {  // the waves share the groups
    const int part = d / groups, waves = nt / WAVE, per = max(1, waves / groups), lane = tid & (WAVE - 1);
    float* inv_of = row + (d + 3) / 4 * 4;  // [groups]
    float* sums = inv_of + groups;          // [groups * per]
    __syncthreads();
    for (int i = tid / WAVE; i < groups * per; i += waves) {
      const float* src = row + i / per * part;
      float s2 = 0.f;
      for (int c = i % per * WAVE + lane; c < part; c += per * WAVE) s2 = fmaf(src[c], src[c], s2);
      s2 = wave_reduce_sum(s2);
      if (lane == 0) sums[i] = s2;
    }
    __syncthreads();
    for (int g = tid; g < groups; g += nt) {
      float s2 = 0.f;
      for (int i = 0; i < per; ++i) s2 += sums[g * per + i];
      inv_of[g] = 1.f / sqrtf(s2 / part + eps);
    }
    __syncthreads();
    const bool quads = by4 && part % 4 == 0;
    if (quads) {
      for (int c = tid * 4; c < d; c += nt * 4) {
        f32x4 v = load4(row + c);
        const f32x4 g = load4(w + c);
        const float inv = inv_of[c / part];
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] *= inv * g[e];
        store4(h + t * dp + c, v);
      }
    }
    for (int c = quads ? d + tid : tid; c < dp; c += nt)
      store_f32(h + t * dp + c, c < d ? row[c] * inv_of[c / part] * w[c] : 0.f);
    return;
  }
  ss = wave_reduce_sum(ss);
  if ((tid & (WAVE - 1)) == 0) red[tid / WAVE] = ss;
  __syncthreads();
  ss = 0.f;
  for (int i = 0; i < nt / WAVE; ++i) ss += red[i];
  const float inv = 1.f / sqrtf(ss / d + eps);
  if (by4) {
    for (int c = tid * 4; c < d; c += nt * 4) {
      f32x4 v = load4(row + c);
      const f32x4 g = load4(w + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] *= inv * g[e];
      store4(h + t * dp + c, v);
    }
  }
  for (int c = by4 ? d + tid : tid; c < dp; c += nt) store_f32(h + t * dp + c, c < d ? row[c] * inv * w[c] : 0.f);
}

// 64 columns x 16 groups of splits per workgroup
__global__ __launch_bounds__(1024) void residual_sum_kernel(
    const float* __restrict__ partials,  // [n_splits, batch, n]
    const float* __restrict__ bias, float* __restrict__ x, long x_stride, int n_splits, int batch, int n, int d,
    float mult) {
  __shared__ float acc[16][64];
  const int ol = threadIdx.x & 63, sg = threadIdx.x >> 6;
  const int c = blockIdx.x * 64 + ol, b = blockIdx.y;
  float v = 0.f;
  if (c < d)
    for (int s = sg; s < n_splits; s += 16) v += partials[((size_t)s * batch + b) * n + c];
  acc[sg][ol] = v;
  __syncthreads();
  if (sg != 0 || c >= d) return;
  float sum = bias ? bias[c] : 0.f;
#pragma unroll
  for (int k = 0; k < 16; ++k) sum += acc[k][ol];
  x[(size_t)b * x_stride + c] = fmaf(mult, sum, x[(size_t)b * x_stride + c]);
}

template <typename T>
__global__ __launch_bounds__(256) void bias_relu2_kernel(T* __restrict__ y, const float* __restrict__ bias, int n, long total) {
  const long i = ((long)blockIdx.x * 256 + threadIdx.x) * 8;
  if (i >= total) return;  // n % 8 == 0: a group of 8 never crosses a row
  const int c = i % n;
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const float v = fmaxf(load_f32(y + i + e) + bias[c + e], 0.f);
    store_f32(y + i + e, v * v);
  }
}

// z > 0: pos z^2 + z/2;  z <= 0: neg (exp(z) - 1 - z) + z/2
struct XieluConstants {
  float pos, neg;
};

__device__ __forceinline__ float xielu(const XieluConstants& k, float z) {
  const float low = fminf(z, 0.f);
  // exp(z) - 1 - z; near 0 by its series, which does not cancel
  float r = expf(low) - 1.f - low;
  if (low > -0.5f) {
    float t = 1.f / 362880.f;
    t = fmaf(t, low, 1.f / 40320.f);
    t = fmaf(t, low, 1.f / 5040.f);
    t = fmaf(t, low, 1.f / 720.f);
    t = fmaf(t, low, 1.f / 120.f);
    t = fmaf(t, low, 1.f / 24.f);
    t = fmaf(t, low, 1.f / 6.f);
    t = fmaf(t, low, 0.5f);
    r = t * low * low;
  }
  return fmaf(0.5f, z, z > 0.f ? k.pos * z * z : k.neg * r);
}

template <typename T>
__global__ __launch_bounds__(256) void bias_xielu_kernel(
    T* __restrict__ y, const float* __restrict__ bias, int n, long total, XieluConstants k) {
  const long i = ((long)blockIdx.x * 256 + threadIdx.x) * 8;
  if (i >= total) return;  // n % 8 == 0: a group of 8 never crosses a row
  const int c = i % n;
  float v[8], b[8];
  load8(y + i, v);
  load8(bias + c, b);
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = xielu(k, v[e] + b[e]);
  store8(y + i, v);
}

// 64 columns x 16 groups of splits per workgroup
__global__ __launch_bounds__(1024) void sum_xielu_kernel(
    const float* __restrict__ partials,  // [n_splits, batch, n]
    const float* __restrict__ bias, float* __restrict__ out, int n_splits, int batch, int n, XieluConstants k) {
  __shared__ float acc[16][64];
  const int ol = threadIdx.x & 63, sg = threadIdx.x >> 6;
  const int c = blockIdx.x * 64 + ol, b = blockIdx.y;
  float v = 0.f;
  if (c < n)
    for (int s = sg; s < n_splits; s += 16) v += partials[((size_t)s * batch + b) * n + c];
  acc[sg][ol] = v;
  __syncthreads();
  if (sg != 0 || c >= n) return;
  float sum = bias[c];
#pragma unroll
  for (int s = 0; s < 16; ++s) sum += acc[s][ol];
  out[(size_t)b * n + c] = xielu(k, sum);
}

// ------------------------------------------------------------------- host

static bool wide(const torch::Tensor& t) {
  TORCH_CHECK(t.is_cuda() && (t.dtype() == torch::kFloat32 || t.dtype() == torch::kBFloat16));
  return t.dtype() == torch::kFloat32;
}

static const float* vec(const c10::optional<torch::Tensor>& t, int64_t n) {
  if (!t.has_value()) return nullptr;
  TORCH_CHECK(t->is_cuda() && t->dtype() == torch::kFloat32 && t->is_contiguous() && t->numel() >= n);
  return t->data_ptr<float>();
}

// x [T, >= d] f32, updated in place if y [T, >= d] or [parts, T, >= d] is given; returns the norm [T, dp] of `groups` equal parts, or
// nothing if w is absent
torch::Tensor residual_norm(torch::Tensor x, c10::optional<torch::Tensor> y, c10::optional<torch::Tensor> bias,
                            c10::optional<torch::Tensor> w, int64_t d, double eps, bool out_f32, double mult,
                            int64_t groups) {
  TORCH_CHECK(x.is_cuda() && x.dtype() == torch::kFloat32 && x.dim() == 2 && x.stride(1) == 1 && x.size(1) >= d);
  TORCH_CHECK(groups >= 1 && d % groups == 0, d, " values in ", groups, " groups");
  const long t = x.size(0), dp = w.has_value() ? (d + 7) / 8 * 8 : 0;
  bool yf = true;
  const void* yp = nullptr;
  long ys = 0, part_stride = 0;
  int parts = 1;
  if (y.has_value()) {
    yf = wide(*y);
    TORCH_CHECK((y->dim() == 2 || y->dim() == 3) && y->stride(-1) == 1 && y->size(-2) == t && y->size(-1) >= d);
    yp = y->data_ptr();
    ys = y->stride(-2);
    if (y->dim() == 3) {
      parts = y->size(0);
      part_stride = y->stride(0);
      TORCH_CHECK(parts >= 1);
    }
  }
  const float* bp = vec(bias, d);
  const float* wp = vec(w, d);
  auto h = torch::empty({wp ? t : 0, dp}, x.options().dtype(out_f32 ? torch::kFloat32 : torch::kBFloat16));
  if (t == 0) return h;
  const size_t lds = d * 4 + (groups > 1 ? (2 * groups + 16 + 4) * 4 : 0);
  TORCH_CHECK(lds <= 65536 - 64, "width ", d, " in ", groups, " groups is not supported");
  const int threads = t < 512 ? 1024 : 256;
  auto aligned = [](const void* p, int bytes) { return reinterpret_cast<uintptr_t>(p) % bytes == 0; };
  const bool by4 = d % 4 == 0 && x.stride(0) % 4 == 0 && ys % 4 == 0 && part_stride % 4 == 0 && aligned(x.data_ptr(), 16) &&
                   aligned(yp, yf ? 16 : 8) && aligned(bp, 16) && aligned(wp, 16);
  auto stream = at::cuda::getCurrentCUDAStream();
#define RN(TY, TH)                                                                                          \
  residual_norm_kernel<TY, TH><<<t, threads, lds, stream>>>(                                                \
      x.data_ptr<float>(), x.stride(0), reinterpret_cast<const TY*>(yp), ys, bp, wp, (float)eps,            \
      wp ? reinterpret_cast<TH*>(h.data_ptr()) : nullptr, (int)d, (int)dp, by4, (float)mult, (int)groups, parts, part_stride)
  if (yf && out_f32) RN(float, float);
  else if (yf) RN(float, unsigned short);
  else if (out_f32) RN(unsigned short, float);
  else RN(unsigned short, unsigned short);
#undef RN
  HIP_CHECK_LAST();
  return h;
}

// partials [splits, T, >= d] of gemv_bf16's raw mode
void residual_sum(torch::Tensor partials, c10::optional<torch::Tensor> bias, torch::Tensor x, int64_t d,
                  double mult) {
  TORCH_CHECK(partials.is_cuda() && partials.dtype() == torch::kFloat32 && partials.dim() == 3 && partials.is_contiguous());
  TORCH_CHECK(x.is_cuda() && x.dtype() == torch::kFloat32 && x.dim() == 2 && x.stride(1) == 1);
  const int batch = partials.size(1), n = partials.size(2);
  TORCH_CHECK(x.size(0) == batch && x.size(1) >= d && n >= d && batch <= 65535);
  if (batch == 0) return;
  residual_sum_kernel<<<dim3((d + 63) / 64, batch), 1024, 0, at::cuda::getCurrentCUDAStream()>>>(
      partials.data_ptr<float>(), vec(bias, d), x.data_ptr<float>(), x.stride(0), (int)partials.size(0), batch, n, (int)d,
      (float)mult);
  HIP_CHECK_LAST();
}

// in place
torch::Tensor bias_relu2(torch::Tensor y, torch::Tensor bias) {
  const bool f = wide(y);
  TORCH_CHECK(y.dim() == 2 && y.is_contiguous() && y.size(1) % 8 == 0);
  const float* bp = vec(bias, y.size(1));
  const long total = y.numel();
  if (total == 0) return y;
  const long blocks = (total / 8 + 255) / 256;
  auto stream = at::cuda::getCurrentCUDAStream();
  if (f) {
    bias_relu2_kernel<float><<<blocks, 256, 0, stream>>>(y.data_ptr<float>(), bp, (int)y.size(1), total);
  } else {
    bias_relu2_kernel<unsigned short><<<blocks, 256, 0, stream>>>(BF16P(y), bp, (int)y.size(1), total);
  }
  HIP_CHECK_LAST();
  return y;
}

// y [T, n] in place, or partials [splits, T, n] of gemv_bf16's raw mode
torch::Tensor bias_xielu(torch::Tensor y, torch::Tensor bias, double pos, double neg) {
  const bool f = wide(y);
  TORCH_CHECK(y.is_contiguous() && (y.dim() == 2 || (y.dim() == 3 && f)));
  const int n = y.size(-1);
  const float* bp = vec(bias, n);
  const XieluConstants k{(float)pos, (float)neg};
  auto stream = at::cuda::getCurrentCUDAStream();
  if (y.dim() == 3) {
    const int batch = y.size(1);
    TORCH_CHECK(batch <= 65535);
    auto out = torch::empty({batch, n}, y.options());
    if (batch > 0) {
      sum_xielu_kernel<<<dim3((n + 63) / 64, batch), 1024, 0, stream>>>(
          y.data_ptr<float>(), bp, out.data_ptr<float>(), (int)y.size(0), batch, n, k);
    }
    HIP_CHECK_LAST();
    return out;
  }
  TORCH_CHECK(n % 8 == 0 && reinterpret_cast<uintptr_t>(y.data_ptr()) % 16 == 0 && reinterpret_cast<uintptr_t>(bp) % 16 == 0);
  const long total = y.numel();
  if (total == 0) return y;
  const long blocks = (total / 8 + 255) / 256;
  if (f) {
    bias_xielu_kernel<float><<<blocks, 256, 0, stream>>>(y.data_ptr<float>(), bp, n, total, k);
  } else {
    bias_xielu_kernel<unsigned short><<<blocks, 256, 0, stream>>>(BF16P(y), bp, n, total, k);
  }
  HIP_CHECK_LAST();
  return y;
}
