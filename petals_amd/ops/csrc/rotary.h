// Rotation turns the pair (i, i + n/2) of the first n values by p f_i. The angle is
// reduced to a quarter turn in double precision, so that it is exact at any position.
#pragma once

#include "common.h"
#include <torch/extension.h>

struct Rotation {
  const double* quarters;  // [turned / 2] f_i in quarter turns per position
  int turned;              // values that turn; those behind them pass
};

__device__ __forceinline__ void sin_cos(double turns4, float& s, float& c) {
  const double whole = rint(turns4);
  const float x = (float)((turns4 - whole) * 1.5707963267948966), t = x * x;  // |x| <= pi/4: series
  float a = -1.f / 39916800.f, b = 1.f / 479001600.f;
  a = fmaf(a, t, 1.f / 362880.f);
  b = fmaf(b, t, -1.f / 3628800.f);
  a = fmaf(a, t, -1.f / 5040.f);
  b = fmaf(b, t, 1.f / 40320.f);
  a = fmaf(a, t, 1.f / 120.f);
  b = fmaf(b, t, -1.f / 720.f);
  a = fmaf(a, t, -1.f / 6.f);
  b = fmaf(b, t, 1.f / 24.f);
  b = fmaf(b, t, -0.5f);
  const float sx = fmaf(a * t, x, x), cx = fmaf(b, t, 1.f);
  const int q = (int)((long)whole & 3);
  s = q & 1 ? cx : sx;
  c = q & 1 ? sx : cx;
  if (q & 2) s = -s;
  if (q == 1 || q == 2) c = -c;
}

static Rotation rotation(const torch::Tensor& quarters) {
  TORCH_CHECK(quarters.is_cuda() && quarters.dtype() == torch::kFloat64 && quarters.is_contiguous());
  return Rotation{quarters.data_ptr<double>(), 2 * (int)quarters.numel()};
}
