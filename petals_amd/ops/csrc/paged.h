// Rows of a ragged batch over a paged cache, shared by the kernels that read it.
#pragma once

#include "common.h"
#include <torch/extension.h>

using bf16x8 = __attribute__((ext_vector_type(8))) short;
using f32x4 = __attribute__((ext_vector_type(4))) float;

#define PAGE 64  // tokens per page
#define BF16P(t) reinterpret_cast<unsigned short*>((t).data_ptr())

struct PagedRows {
  const int* pos;     // [T] position of each row
  const int* owner;   // [T] sequence of each row
  const int* tables;  // [S, width] pages of each sequence
  int width;
  int num_pages;
};

// start of the cache row of (sequence, key) in tokens, -1 if there is none
static __device__ __forceinline__ long cache_row(const PagedRows& b, int seq, int key) {
  const int slot = key / PAGE;
  if (key < 0 || slot >= b.width) return -1;
  const int page = b.tables[(size_t)seq * b.width + slot];
  if (page < 0 || page >= b.num_pages) return -1;
  return (long)page * PAGE + (key - slot * PAGE);
}

template <typename T> __device__ __forceinline__ float load_f32(const T* p);
template <> __device__ __forceinline__ float load_f32<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float load_f32<unsigned short>(const unsigned short* p) { return bf16_to_f32(*p); }
template <typename T> __device__ __forceinline__ void store_f32(T* p, float v);
template <> __device__ __forceinline__ void store_f32<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void store_f32<unsigned short>(unsigned short* p, float v) { *p = f32_to_bf16(v); }

// 8 consecutive elements, 16-byte aligned
static __device__ __forceinline__ void load8(const float* p, float* v) {
#pragma unroll
  for (int h = 0; h < 2; ++h) {
    const f32x4 a = reinterpret_cast<const f32x4*>(p)[h];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[4 * h + e] = a[e];
  }
}
static __device__ __forceinline__ void load8(const unsigned short* p, float* v) {
  const bf16x8 a = *reinterpret_cast<const bf16x8*>(p);
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = bf16_to_f32((unsigned short)a[e]);
}
static __device__ __forceinline__ void store8(float* p, const float* v) {
#pragma unroll
  for (int h = 0; h < 2; ++h)
    reinterpret_cast<f32x4*>(p)[h] = f32x4{v[4 * h], v[4 * h + 1], v[4 * h + 2], v[4 * h + 3]};
}
static __device__ __forceinline__ void store8(unsigned short* p, const float* v) {
  bf16x8 a;
#pragma unroll
  for (int e = 0; e < 8; ++e) a[e] = (short)f32_to_bf16(v[e]);
  *reinterpret_cast<bf16x8*>(p) = a;
}

using v4s = __attribute__((ext_vector_type(4))) short;

// PV B-fragment: keys hi*8..hi*8+7 of one dim per lane, read from the row-major
// tile by two transposing LDS loads. p: row hi*8 + (lane&15)/4, column
// 4*(lane&3) of a 16-wide dim block; after the load lane i holds column i.
static __device__ __forceinline__ bf16x8 load_keys(const unsigned short* p, int row_elems) {
  using lds_v4s = __attribute__((address_space(3))) v4s;
  const v4s a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s*)p);
  const v4s b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s*)(p + 4 * row_elems));
  return bf16x8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}

static PagedRows paged_rows(const torch::Tensor& pos, const torch::Tensor& owner, const torch::Tensor& tables,
                            const torch::Tensor& cache, int64_t tokens) {
  TORCH_CHECK(cache.is_cuda() && cache.dim() == 3 && cache.size(1) == PAGE && cache.is_contiguous(),
              "the cache must be [pages, ", PAGE, ", width]");
  for (const auto& t : {pos, owner, tables})
    TORCH_CHECK(t.is_cuda() && t.dtype() == torch::kInt32 && t.is_contiguous(), "int32 device metadata expected");
  TORCH_CHECK(pos.numel() == tokens && owner.numel() == tokens && tables.dim() == 2, "metadata does not fit the rows");
  return PagedRows{pos.data_ptr<int>(), owner.data_ptr<int>(), tables.data_ptr<int>(),
                   (int)tables.size(1), (int)cache.size(0)};
}
