// Sublayer kernels for blocks that norm each sublayer's OUTPUT and keep the
// residual stream in 32-bit (CDNA4, gfx950).
//
//   sublayer_out      sum of a token's (weighted) sublayer rows -> RMS norm with
//                     a zero-centered weight -> + residual, and, for a sublayer
//                     that is followed by routed experts, the 32-bit router:
//                     logits, softmax over all experts, top-k
//   batched_linear    out[t, h, n] = sum_k a[t, h, k] w[h, n, k]: the per-head
//                     projections of latent attention, MFMA for bf16 weights
//   clamped_swiglu    g * sigmoid(alpha g) * (u + 1), g and u clamped
//   moe_group         expert-sorted, tile-padded (token, slot) pairs for moe_gemm
//   moe_linear_f32    expert products in 32-bit

#include "common.h"
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>

using bf16x8 = __attribute__((ext_vector_type(8))) short;
using f32x4 = __attribute__((ext_vector_type(4))) float;

#define BF16P(t) reinterpret_cast<unsigned short*>((t).data_ptr())

__device__ __forceinline__ float ld(const float* p) { return *p; }
__device__ __forceinline__ float ld(const unsigned short* p) { return bf16_to_f32(*p); }
__device__ __forceinline__ void st(float* p, float v) { *p = v; }
__device__ __forceinline__ void st(unsigned short* p, float v) { *p = f32_to_bf16(v); }

// 8 consecutive elements, 16-byte aligned
__device__ __forceinline__ void ld8(const float* p, float* v) {
#pragma unroll
  for (int h = 0; h < 2; ++h) {
    const f32x4 a = reinterpret_cast<const f32x4*>(p)[h];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[4 * h + e] = a[e];
  }
}
__device__ __forceinline__ void ld8(const unsigned short* p, float* v) {
  const bf16x8 a = *reinterpret_cast<const bf16x8*>(p);
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = bf16_to_f32((unsigned short)a[e]);
}

// sum over the workgroup, the same value in every thread; red holds one float
// per wave and is free again on return
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_reduce_sum(v);
  if ((threadIdx.x & (WAVE - 1)) == 0) red[threadIdx.x / WAVE] = v;
  __syncthreads();
  float s = 0.f;
  for (int i = 0; i < (int)blockDim.x / WAVE; ++i) s += red[i];
  __syncthreads();
  return s;
}

// ---------------------------------------------------------- sublayer output

// One workgroup per token.
//   y [T*k, ys]     sublayer rows; a token's k rows are summed with slot_w
//   x [T, dp]       residual before, xo after (null: the norm alone is written)
//   xb              bf16 copy of xo or null
//   router [E, dp]  or null; sel/sel_w [T, top] get the experts and their scores
template <typename TY, typename TW>
__global__ __launch_bounds__(1024) void sublayer_out_kernel(
    const TY* __restrict__ y, int ys, int k, const float* __restrict__ slot_w,
    const float* __restrict__ norm_w, float eps,
    const float* __restrict__ x, float* __restrict__ xo, unsigned short* __restrict__ xb,
    const TW* __restrict__ router, int experts, int top, int* __restrict__ sel, float* __restrict__ sel_w,
    int d, int dp, bool y_wide) {
  extern __shared__ float sm[];
  float* row = sm;          // [dp], dp % 8 == 0
  float* logit = row + dp;  // [experts]
  __shared__ float red[16];
  const int tid = threadIdx.x, nt = blockDim.x;
  const size_t t = blockIdx.x;

  float ss = 0.f;
  for (int c = tid * 8; c < d; c += nt * 8) {
    float v[8], u[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = 0.f;
    for (int j = 0; j < k; ++j) {
      const TY* src = y + (t * k + j) * ys + c;
      const float w = slot_w ? slot_w[t * k + j] : 1.f;
      if (y_wide) {
        ld8(src, u);
      } else {
#pragma unroll
        for (int i = 0; i < 8; ++i) u[i] = c + i < d ? ld(src + i) : 0.f;
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] = fmaf(w, u[i], v[i]);
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      if (c + i >= d) v[i] = 0.f;
      row[c + i] = v[i];
      ss = fmaf(v[i], v[i], ss);
    }
  }
  const float inv = 1.f / sqrtf(block_sum(ss, red) / d + eps);
  for (int c = tid * 4; c < dp; c += nt * 4) {
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (c + i < d) v[i] = row[c + i] * inv * (1.f + norm_w[c + i]);
    if (x) v += *reinterpret_cast<const f32x4*>(x + t * dp + c);
    *reinterpret_cast<f32x4*>(xo + t * dp + c) = v;
    *reinterpret_cast<f32x4*>(row + c) = v;
    if (xb) {
      uint2 w;
      w.x = f32_to_bf16(v[0]) | ((unsigned)f32_to_bf16(v[1]) << 16);
      w.y = f32_to_bf16(v[2]) | ((unsigned)f32_to_bf16(v[3]) << 16);
      *reinterpret_cast<uint2*>(xb + t * dp + c) = w;
    }
  }
  if (!router) return;
  __syncthreads();
  const int wave = tid / WAVE, lane = tid & (WAVE - 1);
  // two experts per wave at a time; row and router are zero between d and dp
  for (int e = wave * 2; e < experts; e += nt / WAVE * 2) {
    const bool both = e + 1 < experts;
    float z0 = 0.f, z1 = 0.f;
    const TW* r0 = router + (size_t)e * dp;
    const TW* r1 = both ? r0 + dp : r0;
#pragma unroll 4
    for (int c = lane * 8; c < dp; c += WAVE * 8) {
      float w0[8], w1[8];
      ld8(r0 + c, w0);
      ld8(r1 + c, w1);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        z0 = fmaf(row[c + i], w0[i], z0);
        z1 = fmaf(row[c + i], w1[i], z1);
      }
    }
    z0 = wave_reduce_sum(z0);
    z1 = wave_reduce_sum(z1);
    if (lane == 0) {
      logit[e] = z0;
      if (both) logit[e + 1] = z1;
    }
  }
  __syncthreads();
  if (wave != 0) return;
  float mx = NEG_SENTINEL;
  for (int e = lane; e < experts; e += WAVE) mx = fmaxf(mx, logit[e]);
  mx = wave_reduce_max(mx);
  float sum = 0.f;
  for (int e = lane; e < experts; e += WAVE) sum += expf(logit[e] - mx);
  sum = wave_reduce_sum(sum);
  for (int j = 0; j < top; ++j) {
    float best = NEG_SENTINEL * 2.f;
    int arg = experts;
    for (int e = lane; e < experts; e += WAVE)
      if (logit[e] > best) {
        best = logit[e];
        arg = e;
      }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
      const float ob = __shfl_xor(best, off, WAVE);
      const int oa = __shfl_xor(arg, off, WAVE);
      if (ob > best || (ob == best && oa < arg)) {
        best = ob;
        arg = oa;
      }
    }
    if (arg >= experts) arg = 0;  // logits that compare with nothing (NaN)
    if (lane == 0) {
      sel[t * top + j] = arg;
      sel_w[t * top + j] = expf(best - mx) / sum;
    }
    if ((arg & (WAVE - 1)) == lane) logit[arg] = NEG_SENTINEL * 3.f;  // taken; this lane alone reads it
  }
}

// ----------------------------------------------------------- batched linear

__device__ __forceinline__ bf16x8 frag8(const unsigned short* p, int k, int k_dim, bool wide) {
  if (wide && k + 8 <= k_dim) return *reinterpret_cast<const bf16x8*>(p + k);
  short v[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = k + e < k_dim ? (short)p[k + e] : (short)0;
  return bf16x8{v[0], v[1], v[2], v[3], v[4], v[5], v[6], v[7]};
}
__device__ __forceinline__ bf16x8 frag8(const float* p, int k, int k_dim, bool wide) {
  short v[8];
  if (wide && k + 8 <= k_dim) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(p + k), b = *reinterpret_cast<const f32x4*>(p + k + 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      v[e] = (short)f32_to_bf16(a[e]);
      v[4 + e] = (short)f32_to_bf16(b[e]);
    }
  } else {
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = k + e < k_dim ? (short)f32_to_bf16(p[k + e]) : (short)0;
  }
  return bf16x8{v[0], v[1], v[2], v[3], v[4], v[5], v[6], v[7]};
}

// A wave computes 64 rows x 64 columns of one head; the waves of a workgroup
// take consecutive tiles (columns first). Fragments come straight from global
// memory; the weights are the MFMA's A operand, so that a lane ends up with 4
// neighbouring columns of one row, and rows leave through LDS in 16-byte stores.
template <typename TA, typename TO>
__global__ __launch_bounds__(256) void batched_linear_kernel(
    const TA* __restrict__ a, long a_t, long a_h,   // strides of rows and heads
    const unsigned short* __restrict__ w,           // [H, N, K]
    TO* __restrict__ out, long o_t, long o_h, int t_dim, int n_dim, int k_dim, int n_tiles, bool a_wide,
    bool w_wide, bool o_wide) {
  constexpr int MT = 4, NT = 4;
  __shared__ TO tile[4][16][16 * NT + 16 / sizeof(TO)];
  const int lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE;
  const int col = lane & 15, hi = lane >> 4;
  const int job = blockIdx.x * 4 + wave;
  const int n0 = job % n_tiles * 16 * NT;
  const int t0 = job / n_tiles * 16 * MT;
  const size_t h = blockIdx.y;
  if (t0 >= t_dim) return;  // no barrier below
  const TA* ap[MT];
  const unsigned short* wp[NT];
  bool a_ok[MT], w_ok[NT];
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int t = t0 + m * 16 + col;
    a_ok[m] = t < t_dim;
    ap[m] = a + (size_t)(a_ok[m] ? t : 0) * a_t + h * a_h;
  }
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int c = n0 + n * 16 + col;
    w_ok[n] = c < n_dim;
    wp[n] = w + (h * n_dim + (w_ok[n] ? c : 0)) * (size_t)k_dim;
  }
  f32x4 acc[MT][NT];
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int n = 0; n < NT; ++n) acc[m][n] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
  for (int k0 = 0; k0 < k_dim; k0 += 32) {
    bf16x8 af[MT], wf[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n)
      wf[n] = w_ok[n] ? frag8(wp[n], k0 + hi * 8, k_dim, w_wide) : bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
    for (int m = 0; m < MT; ++m)
      af[m] = a_ok[m] ? frag8(ap[m], k0 + hi * 8, k_dim, a_wide) : bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int n = 0; n < NT; ++n)
        acc[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[n], af[m], acc[m][n], 0, 0, 0);
  }
  // acc[m][n][r]: row t0 + m*16 + col, column n0 + n*16 + hi*4 + r
  constexpr int PER = 16 / sizeof(TO);  // elements of a 16-byte store
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) st(&tile[wave][col][n * 16 + hi * 4 + r], acc[m][n][r]);
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll
    for (int i = lane; i < 16 * 16 * NT / PER; i += WAVE) {
      const int t = t0 + m * 16 + i / (16 * NT / PER), c = i % (16 * NT / PER) * PER;
      if (t >= t_dim || n0 + c >= n_dim) continue;
      const TO* src = &tile[wave][t - t0 - m * 16][c];
      TO* dst = out + (size_t)t * o_t + h * o_h + n0 + c;
      if (o_wide && n0 + c + PER <= n_dim) {
        *reinterpret_cast<f32x4*>(dst) = *reinterpret_cast<const f32x4*>(src);
      } else {
        for (int e = 0; e < PER && n0 + c + e < n_dim; ++e) dst[e] = src[e];
      }
    }
  }
}

// Few rows (t_dim <= 16): the 4 waves of a workgroup share 16 columns and split
// k, so that even a single token spreads a head over many waves.
template <typename TA, typename TO>
__global__ __launch_bounds__(256) void batched_linear_few_kernel(
    const TA* __restrict__ a, long a_t, long a_h, const unsigned short* __restrict__ w,
    TO* __restrict__ out, long o_t, long o_h, int t_dim, int n_dim, int k_dim, bool a_wide, bool w_wide) {
  __shared__ float part[4][16][17];
  const int lane = threadIdx.x & (WAVE - 1), wave = threadIdx.x / WAVE;
  const int col = lane & 15, hi = lane >> 4;
  const int n0 = blockIdx.x * 16;
  const size_t h = blockIdx.y;
  const bool a_ok = col < t_dim, w_ok = n0 + col < n_dim;
  const TA* ap = a + (size_t)(a_ok ? col : 0) * a_t + h * a_h;
  const unsigned short* wp = w + (h * n_dim + (w_ok ? n0 + col : 0)) * (size_t)k_dim;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k0 = wave * 32; k0 < k_dim; k0 += 128) {
    const bf16x8 wf = w_ok ? frag8(wp, k0 + hi * 8, k_dim, w_wide) : bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
    const bf16x8 af = a_ok ? frag8(ap, k0 + hi * 8, k_dim, a_wide) : bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(af, wf, acc, 0, 0, 0);
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) part[wave][hi * 4 + r][col] = acc[r];
  __syncthreads();
  const int t = threadIdx.x >> 4, c = threadIdx.x & 15;
  if (t < t_dim && n0 + c < n_dim)
    st(out + (size_t)t * o_t + h * o_h + n0 + c,
       (part[0][t][c] + part[1][t][c]) + (part[2][t][c] + part[3][t][c]));
}

__global__ __launch_bounds__(256) void batched_linear_f32_kernel(
    const float* __restrict__ a, long a_t, long a_h, const float* __restrict__ w,
    float* __restrict__ out, long o_t, long o_h, int n_dim, int k_dim) {
  const int n = blockIdx.x * 4 + threadIdx.x / WAVE;  // a wave per output
  if (n >= n_dim) return;
  const int lane = threadIdx.x & (WAVE - 1);
  const float* ap = a + (size_t)blockIdx.y * a_t + blockIdx.z * a_h;
  const float* wp = w + ((size_t)blockIdx.z * n_dim + n) * k_dim;
  float s = 0.f;
  for (int k = lane; k < k_dim; k += WAVE) s = fmaf(ap[k], wp[k], s);
  s = wave_reduce_sum(s);
  if (lane == 0) out[(size_t)blockIdx.y * o_t + blockIdx.z * o_h + n] = s;
}

// -------------------------------------------------------------- activation

template <typename T>
__global__ __launch_bounds__(256) void clamped_swiglu_kernel(
    const T* __restrict__ gu, T* __restrict__ out, int half, long total, float limit, float alpha) {
  const long i = ((long)blockIdx.x * 256 + threadIdx.x) * 8;
  if (i >= total) return;  // half % 8 == 0: a group of 8 never crosses a row
  const long r = i / half;
  const T* g = gu + r * 2 * half + (i - r * half);
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const float gv = fminf(ld(g + e), limit);
    const float uv = fmaxf(fminf(ld(g + half + e), limit), -limit);
    st(out + i + e, gv / (1.f + expf(-alpha * gv)) * (uv + 1.f));
  }
}

// ------------------------------------------------------------ expert groups

// One workgroup. counts -> padded offsets -> scatter; every sorted slot and
// every tile is written. The order of an expert's pairs is not fixed, which no
// result depends on (each pair is a row of its own).
__global__ __launch_bounds__(1024) void moe_group_kernel(
    const int* __restrict__ sel, int pairs, int experts, int mt, int slots,
    int* __restrict__ sorted_pairs, int* __restrict__ tile_expert) {
  extern __shared__ int cnt[];  // [experts] counts, then next free slot
  int* end = cnt + experts;     // [experts] end of the padded segment
  const int tid = threadIdx.x;
  for (int e = tid; e < experts; e += blockDim.x) cnt[e] = 0;
  for (int i = tid; i < slots; i += blockDim.x) sorted_pairs[i] = -1;
  for (int i = tid; i < slots / mt; i += blockDim.x) tile_expert[i] = -1;
  __syncthreads();
  for (int i = tid; i < pairs; i += blockDim.x) {
    const int e = sel[i];
    if (e >= 0 && e < experts) atomicAdd(&cnt[e], 1);
  }
  __syncthreads();
  if (tid == 0) {
    int at = 0;
    for (int e = 0; e < experts; ++e) {
      const int padded = (cnt[e] + mt - 1) / mt * mt;
      cnt[e] = at;
      at += padded;
      end[e] = at;
    }
  }
  __syncthreads();
  for (int e = tid; e < experts; e += blockDim.x)
    for (int i = cnt[e]; i < end[e]; i += mt) tile_expert[i / mt] = e;
  __syncthreads();
  for (int i = tid; i < pairs; i += blockDim.x) {
    const int e = sel[i];
    if (e >= 0 && e < experts) sorted_pairs[atomicAdd(&cnt[e], 1)] = i;
  }
}

__global__ __launch_bounds__(64) void moe_linear_f32_kernel(
    const float* __restrict__ w,  // [E, in, out]
    const float* __restrict__ x,  // [rows / k, in]
    const int* __restrict__ sel,  // [rows]
    float* __restrict__ out,      // [rows, out]
    int experts, int k, int in_dim, int out_dim) {
  const int c = blockIdx.x * 64 + threadIdx.x;
  const int e = sel[blockIdx.y];
  if (c >= out_dim || e < 0 || e >= experts) return;
  const float* wp = w + (size_t)e * in_dim * out_dim + c;
  const float* xr = x + (size_t)(blockIdx.y / k) * in_dim;
  float s = 0.f;
  for (int i = 0; i < in_dim; ++i) s = fmaf(xr[i], wp[(size_t)i * out_dim], s);
  out[(size_t)blockIdx.y * out_dim + c] = s;
}

// -------------------------------------------------------------------- host

static bool is_f32(const torch::Tensor& t) {
  TORCH_CHECK(t.is_cuda() && (t.dtype() == torch::kFloat32 || t.dtype() == torch::kBFloat16));
  return t.dtype() == torch::kFloat32;
}

// Returns (xo [T, dp] f32, xb [T, dp] bf16 or empty, sel [T, top], sel_w [T, top])
std::vector<torch::Tensor> sublayer_out(
    torch::Tensor y,                       // [T*k, ys]
    c10::optional<torch::Tensor> slot_w,   // [T, k] f32
    torch::Tensor norm_w,                  // [d] f32
    double eps,
    c10::optional<torch::Tensor> x,        // [T, dp] f32
    int64_t dp,
    bool want_bf16,
    c10::optional<torch::Tensor> router,   // [E, dp]
    int64_t top) {
  const bool yf = is_f32(y);
  TORCH_CHECK(y.dim() == 2 && y.is_contiguous() && norm_w.is_contiguous() && norm_w.dtype() == torch::kFloat32);
  const int d = norm_w.numel();
  int k = 1;
  long t = y.size(0);
  const float* sw = nullptr;
  if (slot_w.has_value()) {
    TORCH_CHECK(slot_w->is_contiguous() && slot_w->dtype() == torch::kFloat32 && slot_w->dim() == 2);
    k = slot_w->size(1);
    t = slot_w->size(0);
    sw = slot_w->data_ptr<float>();
  }
  TORCH_CHECK(y.size(0) == t * k && y.size(1) >= d && dp >= d && dp % 8 == 0, "sublayer rows do not fit");
  // whole groups of 8 may be read: aligned rows that reach to the next multiple of 8
  const bool y_wide = y.size(1) % 8 == 0 && reinterpret_cast<uintptr_t>(y.data_ptr()) % 16 == 0;
  auto f32o = y.options().dtype(torch::kFloat32);
  auto xo = torch::empty({t, (long)dp}, f32o);
  auto xb = torch::empty({want_bf16 ? t : 0, (long)dp}, y.options().dtype(torch::kBFloat16));
  const float* xp = nullptr;
  if (x.has_value()) {
    TORCH_CHECK(x->is_contiguous() && x->dtype() == torch::kFloat32 && x->size(0) == t && x->size(1) == dp);
    xp = x->data_ptr<float>();
  }
  int experts = 0;
  bool rf = false;
  const void* rp = nullptr;
  if (router.has_value()) {
    rf = is_f32(*router);
    TORCH_CHECK(router->is_contiguous() && router->dim() == 2 && router->size(1) == dp);
    TORCH_CHECK(reinterpret_cast<uintptr_t>(router->data_ptr()) % 16 == 0);
    experts = router->size(0);
    TORCH_CHECK(top >= 1 && top <= experts);
    rp = router->data_ptr();
  }
  auto sel = torch::empty({experts ? t : 0, (long)top}, y.options().dtype(torch::kInt32));
  auto sel_w = torch::empty({experts ? t : 0, (long)top}, f32o);
  const size_t lds = ((size_t)dp + experts) * 4;
  TORCH_CHECK(lds <= 65536 - 64, "width ", d, " with ", experts, " experts is not supported");
  const int threads = t < 64 ? 1024 : 256;
  auto stream = at::cuda::getCurrentCUDAStream();
  unsigned short* xbp = want_bf16 ? BF16P(xb) : nullptr;
  int* selp = experts ? sel.data_ptr<int>() : nullptr;
  float* selwp = experts ? sel_w.data_ptr<float>() : nullptr;
  if (t > 0) {
#define SO(TY, TW, YP)                                                                                     \
  sublayer_out_kernel<TY, TW><<<t, threads, lds, stream>>>(                                                \
      YP, (int)y.size(1), k, sw, norm_w.data_ptr<float>(), (float)eps, xp, xo.data_ptr<float>(), xbp,      \
      reinterpret_cast<const TW*>(rp), experts, (int)top, selp, selwp, d, (int)dp, y_wide)
    if (yf && rf) SO(float, float, y.data_ptr<float>());
    else if (yf) SO(float, unsigned short, y.data_ptr<float>());
    else if (rf) SO(unsigned short, float, BF16P(y));
    else SO(unsigned short, unsigned short, BF16P(y));
#undef SO
    HIP_CHECK_LAST();
  }
  return {xo, xb, sel, sel_w};
}

// a: [T, H, K] view (any row and head stride, unit k stride); w: [H, N, K]
// into: where the result goes, a view [t, h, n] with unit stride in n (default: a new tensor)
torch::Tensor batched_linear(torch::Tensor a, torch::Tensor w, bool out_f32, c10::optional<torch::Tensor> into) {
  const bool af = is_f32(a), wf = is_f32(w);
  TORCH_CHECK(a.dim() == 3 && w.dim() == 3 && w.is_contiguous() && a.stride(2) == 1);
  const long t = a.size(0), h = a.size(1), k = a.size(2), n = w.size(1);
  TORCH_CHECK(w.size(0) == h && w.size(2) == k, "batched_linear shapes");
  TORCH_CHECK(!wf || (af && out_f32), "32-bit weights need 32-bit rows");
  auto out = into.has_value() ? *into
                              : torch::empty({t, h, n}, a.options().dtype(out_f32 ? torch::kFloat32 : torch::kBFloat16));
  TORCH_CHECK(out.is_cuda() && out.dtype() == (out_f32 ? torch::kFloat32 : torch::kBFloat16) && out.dim() == 3 &&
              out.size(0) == t && out.size(1) == h && out.size(2) == n && out.stride(2) == 1, "batched_linear result");
  if (t == 0) return out;
  auto stream = at::cuda::getCurrentCUDAStream();
  const long at_ = a.stride(0), ah = a.stride(1), ot = out.stride(0), oh = out.stride(1);
  if (wf) {
    TORCH_CHECK(t <= 65535 && h <= 65535);
    batched_linear_f32_kernel<<<dim3((n + 3) / 4, t, h), 256, 0, stream>>>(
        a.data_ptr<float>(), at_, ah, w.data_ptr<float>(), out.data_ptr<float>(), ot, oh, n, k);
    HIP_CHECK_LAST();
    return out;
  }
  const size_t ab = af ? 4 : 2;
  const bool a_wide = (reinterpret_cast<uintptr_t>(a.data_ptr()) % 16 == 0) && (at_ * ab) % 16 == 0 && (ah * ab) % 16 == 0;
  const bool w_wide = k % 8 == 0;
  const long ob = out_f32 ? 4 : 2;
  const bool o_wide = ot * ob % 16 == 0 && oh * ob % 16 == 0 && reinterpret_cast<uintptr_t>(out.data_ptr()) % 16 == 0;
  const int n_tiles = (n + 63) / 64;
  const long jobs = n_tiles * ((t + 63) / 64);
#define BL(TA, TO, AP, OP)                                                               \
  batched_linear_kernel<TA, TO><<<dim3((jobs + 3) / 4, h), 256, 0, stream>>>(            \
      AP, at_, ah, BF16P(w), OP, ot, oh, t, n, k, n_tiles, a_wide, w_wide, o_wide)
#define BF(TA, TO, AP, OP)                                                           \
  batched_linear_few_kernel<TA, TO><<<dim3((n + 15) / 16, h), 256, 0, stream>>>(     \
      AP, at_, ah, BF16P(w), OP, ot, oh, t, n, k, a_wide, w_wide)
#define BLO(TA, AP)                                                       \
  do {                                                                    \
    if (t <= 16) {                                                        \
      if (out_f32) BF(TA, float, AP, out.data_ptr<float>());              \
      else BF(TA, unsigned short, AP, BF16P(out));                        \
    } else if (out_f32) BL(TA, float, AP, out.data_ptr<float>());   \
    else BL(TA, unsigned short, AP, BF16P(out));                    \
  } while (0)
  if (af) BLO(float, a.data_ptr<float>()); else BLO(unsigned short, BF16P(a));
#undef BF
#undef BLO
#undef BL
  HIP_CHECK_LAST();
  return out;
}

torch::Tensor clamped_swiglu(torch::Tensor gu, double limit, double alpha) {
  const bool f = is_f32(gu);
  TORCH_CHECK(gu.dim() == 2 && gu.is_contiguous() && gu.size(1) % 16 == 0, "gate|up rows of 2 x (a multiple of 8)");
  const int half = gu.size(1) / 2;
  auto out = torch::empty({gu.size(0), half}, gu.options());
  const long total = out.numel();
  if (total == 0) return out;
  const long blocks = (total / 8 + 255) / 256;
  auto stream = at::cuda::getCurrentCUDAStream();
  if (f)
    clamped_swiglu_kernel<float><<<blocks, 256, 0, stream>>>(
        gu.data_ptr<float>(), out.data_ptr<float>(), half, total, (float)limit, (float)alpha);
  else
    clamped_swiglu_kernel<unsigned short><<<blocks, 256, 0, stream>>>(
        BF16P(gu), BF16P(out), half, total, (float)limit, (float)alpha);
  HIP_CHECK_LAST();
  return out;
}

// sel [R] expert of each (token, slot) pair -> (sorted_pairs, tile_expert), see moe.hip
std::vector<torch::Tensor> moe_group(torch::Tensor sel, int64_t experts, int64_t mt) {
  TORCH_CHECK(sel.is_cuda() && sel.dtype() == torch::kInt32 && sel.is_contiguous());
  TORCH_CHECK(experts >= 1 && experts <= 4096 && mt >= 1);
  const long r = sel.numel();
  // at most min(r, experts) segments end in a partly filled tile
  const long slots = (r + std::min(r, (long)experts) * (mt - 1) + mt - 1) / mt * mt;
  auto pairs = torch::empty({slots}, sel.options());
  auto tiles = torch::empty({slots / mt}, sel.options());
  moe_group_kernel<<<1, 1024, experts * 8, at::cuda::getCurrentCUDAStream()>>>(
      sel.data_ptr<int>(), r, experts, mt, slots, pairs.data_ptr<int>(), tiles.data_ptr<int>());
  HIP_CHECK_LAST();
  return {pairs, tiles};
}

torch::Tensor moe_linear_f32(torch::Tensor w, torch::Tensor x, torch::Tensor sel, int64_t k) {
  TORCH_CHECK(is_f32(w) && is_f32(x) && w.dim() == 3 && x.dim() == 2 && w.is_contiguous() && x.is_contiguous());
  TORCH_CHECK(sel.is_cuda() && sel.dtype() == torch::kInt32 && sel.is_contiguous());
  const long rows = sel.numel();
  TORCH_CHECK(x.size(1) == w.size(1) && x.size(0) * k == rows);
  auto out = torch::empty({rows, w.size(2)}, x.options());
  const long step = std::max(1L, 32768 / k) * k;  // rows per launch (grid.y), whole tokens
  for (long r = 0; r < rows; r += step)
    moe_linear_f32_kernel<<<dim3((w.size(2) + 63) / 64, std::min(step, rows - r)), 64, 0,
                            at::cuda::getCurrentCUDAStream()>>>(
        w.data_ptr<float>(), x.data_ptr<float>() + r / k * w.size(1), sel.data_ptr<int>() + r,
        out.data_ptr<float>() + r * w.size(2), (int)w.size(0), (int)k, (int)w.size(1), (int)w.size(2));
  HIP_CHECK_LAST();
  return out;
}
