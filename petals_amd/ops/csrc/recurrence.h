// Parts shared by the kernels of recurrent layers, whose prompts are cut into
// chunks of CH tokens.
#pragma once

#include "common.h"
#include "paged.h"

#define CH 16  // tokens of a chunk
#define LOG2E 1.4426950408889634f

// max(x, 0) + log1p(u), u = exp(-|x|); log1p(u) = log(w) u / (w - 1) with w = 1 + u
// as it is rounded
__device__ __forceinline__ float softplus_f32(float x) {
  const float u = expf(-fabsf(x));
  float w = 1.f + u;
  asm volatile("" : "+v"(w));  // or fast math would take w - 1 for u
  const float d = w - 1.f;
  return fmaxf(x, 0.f) + (d > 0.f ? logf(w) * (u / d) : u);
}

// Fragments of v_mfma_f32_16x16x4f32: A[m = lane&15][k = lane>>4],
// B[k = lane>>4][n = lane&15], C rows (lane>>4)*4 + r, column lane&15. A C tile
// serves as B of four such products as it is: product r takes k = (lane>>4)*4 + r.
__device__ __forceinline__ f32x4 mma16(const f32x4& a, const f32x4& b, f32x4 c) {
#pragma unroll
  for (int r = 0; r < 4; ++r) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[r], b[r], c, 0, 0, 0);
  return c;
}

// a barrier for data in LDS that leaves loads from memory in flight
__device__ __forceinline__ void lds_barrier() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
  __builtin_amdgcn_s_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
}

static void check_f32(const torch::Tensor& t, int64_t n, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.dtype() == torch::kFloat32 && t.is_contiguous() && t.numel() == n, what);
}
static void check_i32(const torch::Tensor& t, int64_t n, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.dtype() == torch::kInt32 && t.is_contiguous() && t.numel() >= n, what);
}
