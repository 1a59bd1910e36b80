// Rows of a layer whose attention and feed-forward read one projection (CDNA4, gfx950).
//
//   prepare_rows   queries, keys and values: bias, short causal convolution, RMS norm of
//                  the whole query and key projections, rotation; writes the cache. In
//                  the same launch the feed-forward's PolyNorm. Each step may be absent.
//   conv_tail      the convolution's inputs that the next step needs
//
// The convolution's inputs of a sequence are kept in its slot of [slots, taps, columns],
// position p in row p % taps; those ahead of position 0 are zero whatever a slot holds.
// One token per sequence: prepare_rows stores its inputs itself, for it reads other rows
// of the slot. Otherwise conv_tail does when all rows have been read.

#include "common.h"
#include "paged.h"
#include "rotary.h"
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>

struct RowShape {
  int nq, nk, nv;      // padded columns of queries, keys and values, from column 0
  int dk;              // padded size of a query or key vector
  int q_size, k_size;  // values of a projection without padding
  int taps, slots;     // taps 0: no convolution
  __device__ __host__ int columns() const { return nq + nk + nv; }
};

struct RowWeights {
  const float* bias;  // [columns] or null
  const float* conv;  // [taps, columns]
  const float* norm;  // [nq + nk] or null
};

struct PolyPart {
  int at, n, padded;  // columns of the feed-forward's rows
  float a, b, c, e;
};

struct ConvState {
  float* inputs;  // [slots, taps, columns]
  const int* slot;
  bool store;
};

// columns c .. c+7 of row t behind the convolution. back: rows of the same sequence
// right before t in this step, at most taps - 1
template <typename TY>
__device__ __forceinline__ void convolved(
    const TY* __restrict__ y, int stride, const RowShape& s, const RowWeights& w, const ConvState& st, size_t t, int p,
    int slot, int back, int c, float* v) {
  constexpr int NEAR = 3;  // earlier inputs that are loaded together
  const int n = s.columns();
  float bias[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
  load8(y + t * stride + c, v);
  if (w.bias) {
    load8(w.bias + c, bias);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] += bias[e];
  }
  if (s.taps == 0) return;
  float* ring = st.inputs + (size_t)slot * s.taps * n + c;
  if (st.store) store8(ring + (size_t)(p % s.taps) * n, v);
  float x[8], f[NEAR + 1][8];
  load8(w.conv + (size_t)(s.taps - 1) * n + c, f[0]);
  // all from this step, or all from the slot: loads without branches between them, taps that do not exist weigh 0
  const bool rows = back >= s.taps - 1, kept = back == 0 && p >= s.taps - 1;
  if (s.taps <= NEAR + 1 && (rows || kept)) {
    float in[NEAR][8];
#pragma unroll
    for (int j = 1; j <= NEAR; ++j) load8(w.conv + (size_t)max(s.taps - 1 - j, 0) * n + c, f[j]);
    if (rows) {
#pragma unroll
      for (int j = 1; j <= NEAR; ++j) load8(y + (t - min(j, s.taps - 1)) * stride + c, in[j - 1]);
#pragma unroll
      for (int j = 0; j < NEAR; ++j)
#pragma unroll
        for (int e = 0; e < 8; ++e) in[j][e] += bias[e];
    } else {
#pragma unroll
      for (int j = 1; j <= NEAR; ++j) load8(ring + (size_t)((p - min(j, s.taps - 1)) % s.taps) * n, in[j - 1]);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] *= f[0][e];
#pragma unroll
    for (int j = 1; j <= NEAR; ++j)
      if (j < s.taps) {
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = fmaf(f[j][e], in[j - 1][e], v[e]);
      }
    return;
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] *= f[0][e];
  for (int ago = 1; ago < s.taps && ago <= p; ++ago) {
    load8(w.conv + (size_t)(s.taps - 1 - ago) * n + c, f[0]);
    if (ago <= back) {
      load8(y + (t - ago) * stride + c, x);
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] += bias[e];
    } else {
      load8(ring + (size_t)((p - ago) % s.taps) * n, x);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = fmaf(f[0][e], x[e], v[e]);
  }
}

// 8 values as they are stored
template <typename T> struct Packed8;
template <> struct Packed8<unsigned short> {
  bf16x8 v;
  __device__ __forceinline__ void load(const unsigned short* p) { v = *reinterpret_cast<const bf16x8*>(p); }
  __device__ __forceinline__ float operator[](int e) const { return bf16_to_f32((unsigned short)v[e]); }
};
template <> struct Packed8<float> {
  f32x4 v[2];
  __device__ __forceinline__ void load(const float* p) {
    v[0] = reinterpret_cast<const f32x4*>(p)[0];
    v[1] = reinterpret_cast<const f32x4*>(p)[1];
  }
  __device__ __forceinline__ float operator[](int e) const { return v[e >> 2][e & 3]; }
};

// out = a N(z) + b N(z^2) + c N(z^3) + e of one row, N dividing by the root mean square
template <typename T, int NT>
__device__ __forceinline__ void poly_row(const T* __restrict__ z, const PolyPart& k, float eps, T* __restrict__ out) {
  constexpr int KEEP = sizeof(T) == 2 ? 8 : 4;  // groups of 8 that a thread holds on to
  __shared__ float red[3][NT / WAVE];
  const int tid = threadIdx.x, groups = k.padded / 8;
  Packed8<T> kept[KEEP];
  float s2 = 0.f, s4 = 0.f, s6 = 0.f;
  auto count = [&](const Packed8<T>& x) {
#pragma unroll
    for (int e = 0; e < 8; ++e) {  // padding is zero
      const float v = x[e], q = v * v;
      s2 += q;
      s4 = fmaf(q, q, s4);
      s6 = fmaf(q * q, q, s6);
    }
  };
#pragma unroll
  for (int i = 0; i < KEEP; ++i)
    if (tid + i * NT < groups) kept[i].load(z + (size_t)(tid + i * NT) * 8);
#pragma unroll
  for (int i = 0; i < KEEP; ++i)
    if (tid + i * NT < groups) count(kept[i]);
  for (int i = tid + KEEP * NT; i < groups; i += NT) {
    Packed8<T> x;
    x.load(z + (size_t)i * 8);
    count(x);
  }
  s2 = wave_reduce_sum(s2);
  s4 = wave_reduce_sum(s4);
  s6 = wave_reduce_sum(s6);
  if ((tid & (WAVE - 1)) == 0) {
    red[0][tid / WAVE] = s2;
    red[1][tid / WAVE] = s4;
    red[2][tid / WAVE] = s6;
  }
  __syncthreads();
  s2 = s4 = s6 = 0.f;
#pragma unroll
  for (int i = 0; i < NT / WAVE; ++i) {
    s2 += red[0][i];
    s4 += red[1][i];
    s6 += red[2][i];
  }
  const float n = k.n;
  const float a = k.a / sqrtf(s2 / n + eps), b = k.b / sqrtf(s4 / n + eps), c = k.c / sqrtf(s6 / n + eps);
  auto write = [&](int i, const Packed8<T>& x) {
    float v[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = fmaf(fmaf(fmaf(c, x[e], b), x[e], a), x[e], k.e);
    store8(out + (size_t)i * 8, v);
  };
#pragma unroll
  for (int i = 0; i < KEEP; ++i)
    if (tid + i * NT < groups) write(tid + i * NT, kept[i]);
  for (int i = tid + KEEP * NT; i < groups; i += NT) {
    Packed8<T> x;
    x.load(z + (size_t)i * 8);
    write(i, x);
  }
}

// Grid: (rows, parts); a part is the queries, the keys, the values or the feed-forward
// of a token. With `spread`, the rows in 8 runs, one for each chiplet, to which
// workgroups are dealt in turn: a row is an input of the next rows' convolution.
template <typename TY, typename TC, int NT>
__global__ __launch_bounds__(NT) void prepare_rows_kernel(
    const TY* __restrict__ y, int stride, RowShape s, RowWeights w, ConvState st, Rotation rot, float turn_factor,
    PagedRows b, TC* __restrict__ q, TC* __restrict__ cache, float eps, PolyPart poly, TY* __restrict__ act,
    long act_stride, int rows, bool spread) {
  extern __shared__ __attribute__((aligned(16))) float row[];  // [columns of the part], then cos and sin of each pair
  __shared__ float red[NT / WAVE];
  const int tid = threadIdx.x, part = blockIdx.y;
  const int ti = spread ? (blockIdx.x & 7) * (gridDim.x >> 3) + (blockIdx.x >> 3) : blockIdx.x;
  if (ti >= rows) return;
  const size_t t = ti;
  if (part == 3) {
    poly_row<TY, NT>(y + t * stride + poly.at, poly, eps, act + t * act_stride);
    return;
  }
  const int seq = b.owner[t], p = b.pos[t];
  int back = 0, slot = 0;
  if (s.taps > 0) {
    while (back < s.taps - 1 && back < ti && b.owner[ti - back - 1] == seq) ++back;
    if (st.slot) slot = min(max(st.slot[seq], 0), s.slots - 1);
  }
  const int width = s.nk + s.nv;
  const long at = part > 0 ? cache_row(b, seq, p) : 0;
  float v[8];
  if (part == 2) {
    for (int c = tid * 8; c < s.nv; c += NT * 8) {
      convolved(y, stride, s, w, st, t, p, slot, back, s.nq + s.nk + c, v);
      if (at >= 0) store8(cache + (size_t)at * width + s.nk + c, v);
    }
    return;
  }
  const int n = part == 0 ? s.nq : s.nk, first = part == 0 ? 0 : s.nq, half = rot.turned / 2;
  float* cs = row + n;
  float* sn = cs + half;
  for (int i = tid; i < half; i += NT) {
    float si, co;
    sin_cos(p * rot.quarters[i], si, co);
    cs[i] = co * turn_factor;
    sn[i] = si * turn_factor;
  }
  float ss = 0.f;
  for (int c = tid * 8; c < n; c += NT * 8) {
    convolved(y, stride, s, w, st, t, p, slot, back, first + c, v);
    if (w.norm) {
      float g[8];
      load8(w.norm + first + c, g);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        ss = fmaf(v[e], v[e], ss);
        v[e] *= g[e];
      }
    }
    store8(row + c, v);
  }
  ss = wave_reduce_sum(ss);
  if ((tid & (WAVE - 1)) == 0) red[tid / WAVE] = ss;
  __syncthreads();
  float inv = 1.f;
  if (w.norm) {
    ss = 0.f;
#pragma unroll
    for (int i = 0; i < NT / WAVE; ++i) ss += red[i];
    inv = 1.f / sqrtf(ss / (part == 0 ? s.q_size : s.k_size) + eps);
  }
  if (at < 0) return;
  TC* dst = part == 0 ? q + t * n : cache + (size_t)at * width;
  const bool by8 = (half & 7) == 0;
  for (int c = tid * 8; c < n; c += NT * 8) {
    const int d = c % s.dk;
    load8(row + c, v);
    if (by8) {
      if (d < 2 * half) {
        const bool low = d < half;
        float o[8], co[8], si[8];
        load8(row + c + (low ? half : -half), o);
        load8(cs + (low ? d : d - half), co);
        load8(sn + (low ? d : d - half), si);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = fmaf(v[e], co[e], low ? -o[e] * si[e] : o[e] * si[e]);
      }
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int i = d + e;
        if (i < half) v[e] = v[e] * cs[i] - row[c + e + half] * sn[i];
        else if (i < 2 * half) v[e] = fmaf(v[e], cs[i - half], row[c + e - half] * sn[i - half]);
      }
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] *= inv;
    store8(dst + c, v);
  }
}

// one workgroup per row
template <typename T, int NT>
__global__ __launch_bounds__(NT) void poly_kernel(
    const T* __restrict__ y, int stride, float eps, PolyPart poly, T* __restrict__ act, long act_stride) {
  const size_t t = blockIdx.x;
  poly_row<T, NT>(y + t * stride + poly.at, poly, eps, act + t * act_stride);
}

// ------------------------------------------------------------ prompts' rows

#define TILE_ROWS 4

// columns c .. c+7 of TILE_ROWS rows from t behind the convolution, whose inputs all are rows of this step
template <int TAPS>
__device__ __forceinline__ void convolved_rows(
    const unsigned short* __restrict__ y, int stride, const RowShape& s, const RowWeights& w, size_t t, int c,
    float (&v)[TILE_ROWS][8]) {
  constexpr int AHEAD = TAPS > 0 ? TAPS - 1 : 0;
  Packed8<unsigned short> in[TILE_ROWS + AHEAD];
#pragma unroll
  for (int r = 0; r < TILE_ROWS + AHEAD; ++r) in[r].load(y + (t + r - AHEAD) * stride + c);
  float bias[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
  if (w.bias) load8(w.bias + c, bias);
  if (TAPS == 0) {
#pragma unroll
    for (int r = 0; r < TILE_ROWS; ++r)
#pragma unroll
      for (int e = 0; e < 8; ++e) v[r][e] = in[r][e] + bias[e];
    return;
  }
#pragma unroll
  for (int r = 0; r < TILE_ROWS; ++r)
#pragma unroll
    for (int e = 0; e < 8; ++e) v[r][e] = 0.f;
#pragma unroll
  for (int j = 0; j < TAPS; ++j) {
    float f[8];
    load8(w.conv + (size_t)j * s.columns() + c, f);
#pragma unroll
    for (int r = 0; r < TILE_ROWS; ++r)
#pragma unroll
      for (int e = 0; e < 8; ++e) v[r][e] = fmaf(f[e], in[r + j][e] + bias[e], v[r][e]);
  }
}

// As prepare_rows_kernel, for TILE_ROWS rows at once: weights and a row's inputs are read
// once for all of them, and nothing but sums and angles leaves the registers. A thread has
// two groups of 8 columns that are rotated with each other (or pass). Needs half % 8 == 0
// and a part of at most 16 NT columns. Grid: (tiles, queries / keys / values).
template <int TAPS, int NT>
__global__ __launch_bounds__(NT) void prepare_tile_kernel(
    const unsigned short* __restrict__ y, int stride, RowShape s, RowWeights w, ConvState st, Rotation rot,
    float turn_factor, PagedRows b, unsigned short* __restrict__ q, unsigned short* __restrict__ cache, float eps,
    int rows) {
  constexpr int R = TILE_ROWS;
  extern __shared__ __attribute__((aligned(16))) float table[];  // [R][2][half]
  __shared__ float red[R][NT / WAVE];
  const int tid = threadIdx.x, part = blockIdx.y, waves = blockDim.x / WAVE;
  const int tile = (blockIdx.x & 7) * (gridDim.x >> 3) + (blockIdx.x >> 3);
  const int t0 = tile * R, live = min(R, rows - t0);
  if (live <= 0) return;
  int p[R], seq[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    p[r] = b.pos[t0 + min(r, live - 1)];
    seq[r] = b.owner[t0 + min(r, live - 1)];
  }
  const bool straight = live == R && seq[0] == seq[R - 1] &&
                        (TAPS == 0 || (t0 >= TAPS - 1 && b.owner[max(t0 - TAPS + 1, 0)] == seq[0]));
  auto columns = [&](int c, float (&v)[R][8]) {
    if (straight) {
      convolved_rows<TAPS>(y, stride, s, w, t0, c, v);
      return;
    }
    float bias[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (w.bias) load8(w.bias + c, bias);
#pragma unroll
    for (int r = 0; r < R; ++r) {  // rows at a sequence's edge
      const int t = t0 + min(r, live - 1);
      const float* ring = nullptr;
      if (TAPS > 0) ring = st.inputs + (size_t)min(max(st.slot[seq[r]], 0), s.slots - 1) * TAPS * s.columns() + c;
#pragma unroll
      for (int e = 0; e < 8; ++e) v[r][e] = 0.f;
#pragma unroll 1
      for (int ago = 0; ago < max(TAPS, 1) && ago <= p[r]; ++ago) {
        float x[8], f[8];
        if (ago <= t && b.owner[t - ago] == seq[r]) {
          load8(y + (size_t)(t - ago) * stride + c, x);
#pragma unroll
          for (int e = 0; e < 8; ++e) x[e] += bias[e];
        } else {
          load8(ring + (size_t)((p[r] - ago) % max(TAPS, 1)) * s.columns(), x);
        }
        if (TAPS > 0) load8(w.conv + (size_t)(TAPS - 1 - ago) * s.columns() + c, f);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[r][e] = TAPS > 0 ? fmaf(f[e], x[e], v[r][e]) : x[e];
      }
    }
  };
  const int width = s.nk + s.nv;
  float v[2][R][8];
  if (part == 2) {
    for (int c = tid * 8; c < s.nv; c += blockDim.x * 8) {
      columns(s.nq + s.nk + c, v[0]);
#pragma unroll
      for (int r = 0; r < R; ++r)
        if (r < live) {
          const long at = cache_row(b, seq[r], p[r]);
          if (at >= 0) store8(cache + (size_t)at * width + s.nk + c, v[0][r]);
        }
    }
    return;
  }
  const int n = part == 0 ? s.nq : s.nk, first = part == 0 ? 0 : s.nq, half = rot.turned / 2;
  const bool busy = tid < n / 16;
  const int head = tid / (s.dk / 16), unit = tid - head * (s.dk / 16);
  const bool turns = unit < half / 8;
  const int d0 = turns ? unit * 8 : 2 * half + (unit - half / 8) * 16;
  const int c0 = head * s.dk + d0, c1 = c0 + (turns ? half : 8);
  float ss[R];
#pragma unroll
  for (int r = 0; r < R; ++r) ss[r] = 0.f;
  if (busy) {
    columns(first + c0, v[0]);
    columns(first + c1, v[1]);
    if (w.norm) {
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        float g[8];
        load8(w.norm + first + (i ? c1 : c0), g);
#pragma unroll
        for (int r = 0; r < R; ++r)
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            ss[r] = fmaf(v[i][r][e], v[i][r][e], ss[r]);
            v[i][r][e] *= g[e];
          }
      }
    }
  }
  for (int i = tid; i < R * half; i += blockDim.x) {
    const int r = i / half, d = i - r * half;
    float si, co;
    sin_cos((straight ? p[0] + r : b.pos[t0 + min(r, live - 1)]) * rot.quarters[d], si, co);
    table[r * 2 * half + d] = co * turn_factor;
    table[r * 2 * half + half + d] = si * turn_factor;
  }
#pragma unroll
  for (int r = 0; r < R; ++r) {
    ss[r] = wave_reduce_sum(ss[r]);
    if ((tid & (WAVE - 1)) == 0) red[r][tid / WAVE] = ss[r];
  }
  __syncthreads();
  if (!busy) return;
#pragma unroll
  for (int r = 0; r < R; ++r) {
    if (r >= live) break;
    float inv = 1.f;
    if (w.norm) {
      float sum = 0.f;
      for (int i = 0; i < waves; ++i) sum += red[r][i];
      inv = 1.f / sqrtf(sum / (part == 0 ? s.q_size : s.k_size) + eps);
    }
    if (turns) {
      float co[8], si[8];
      load8(table + r * 2 * half + d0, co);
      load8(table + r * 2 * half + half + d0, si);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float x = v[0][r][e], z = v[1][r][e];
        v[0][r][e] = x * co[e] - z * si[e];
        v[1][r][e] = fmaf(z, co[e], x * si[e]);
      }
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int e = 0; e < 8; ++e) v[i][r][e] *= inv;
    unsigned short* dst;
    if (part == 0) {
      dst = q + (size_t)(t0 + r) * n;
    } else {
      const long at = cache_row(b, seq[r], p[r]);
      if (at < 0) continue;
      dst = cache + (size_t)at * width;
    }
    store8(dst + c0, v[0][r]);
    store8(dst + c1, v[1][r]);
  }
}

// Grid: (sequences, groups of 2048 columns)
template <typename TY>
__global__ __launch_bounds__(256) void conv_tail_kernel(
    const TY* __restrict__ y, int stride, RowShape s, const float* __restrict__ bias, ConvState st,
    const int* __restrict__ pos, const int* __restrict__ tiles, const int* __restrict__ bounds) {
  const int seq = blockIdx.x, c = (blockIdx.y * 256 + threadIdx.x) * 8;
  if (c >= s.columns() || bounds[seq] >= bounds[seq + 1]) return;
  const int slot = min(max(st.slot[seq], 0), s.slots - 1);
  const int first = tiles[2 * bounds[seq]], last = bounds[seq + 1] - 1;
  const int end = tiles[2 * last] + tiles[2 * last + 1];
  for (int r = max(first, end - s.taps); r < end; ++r) {
    float v[8];
    load8(y + (size_t)r * stride + c, v);
    if (bias) {
      float u[8];
      load8(bias + c, u);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] += u[e];
    }
    store8(st.inputs + ((size_t)slot * s.taps + pos[r] % s.taps) * s.columns() + c, v);
  }
}

// ------------------------------------------------------------------- host

static bool f32_rows(const torch::Tensor& t) {
  TORCH_CHECK(t.is_cuda() && (t.dtype() == torch::kFloat32 || t.dtype() == torch::kBFloat16));
  return t.dtype() == torch::kFloat32;
}

static const float* opt(const c10::optional<torch::Tensor>& t, int64_t n) {
  if (!t.has_value()) return nullptr;
  TORCH_CHECK(t->is_cuda() && t->dtype() == torch::kFloat32 && t->is_contiguous() && t->numel() == n);
  TORCH_CHECK(reinterpret_cast<uintptr_t>(t->data_ptr()) % 16 == 0);
  return t->data_ptr<float>();
}

static void conv_tail(const torch::Tensor& y, const RowShape& s, const RowWeights& w, const ConvState& st, bool single,
                      const torch::Tensor& pos, const c10::optional<torch::Tensor>& tiles,
                      const c10::optional<torch::Tensor>& bounds) {
  if (s.taps <= 1 || single) return;
  const dim3 grid(bounds->numel() - 1, (s.columns() / 8 + 255) / 256);
  auto stream = at::cuda::getCurrentCUDAStream();
#define CT(TY)                                                                                                        \
  conv_tail_kernel<TY><<<grid, 256, 0, stream>>>(reinterpret_cast<const TY*>(y.data_ptr()), (int)y.size(1), s, w.bias, st, \
                                                 pos.data_ptr<int>(), tiles->data_ptr<int>(), bounds->data_ptr<int>())
  if (y.dtype() == torch::kFloat32) CT(float);
  else CT(unsigned short);
#undef CT
  HIP_CHECK_LAST();
}

// y [T, ys]: columns of `heads` query vectors of dk values, kv_heads key vectors, `values` value
// columns. Returns the queries [T, heads * dk] in the cache's dtype; keys and values go to the cache.
//   bias [columns], conv_w [taps, columns], norm [query and key columns], each f32 or absent; dim: values of
//   a vector without padding
//   quarters [pairs] f64: quarter turns per position; turn_factor: of what is turned
//   conv [slots, taps, columns] f32 and slot: absent if there is nothing to remember; single: one row per sequence,
//   else tiles, bounds: the sequences' rows
//   poly: (a, b, c, e) and columns [poly_at, poly_at + ff) of y go through PolyNorm to act [T, padded], a multiple
//   of 8; y has as many columns, zero behind the first ff; empty: none
torch::Tensor prepare_rows(
    torch::Tensor y, torch::Tensor cache, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables, int64_t heads,
    int64_t kv_heads, int64_t dk, int64_t dim, int64_t values, c10::optional<torch::Tensor> bias,
    c10::optional<torch::Tensor> conv_w, c10::optional<torch::Tensor> norm, torch::Tensor quarters, double turn_factor,
    c10::optional<torch::Tensor> conv, c10::optional<torch::Tensor> slot, bool single,
    c10::optional<torch::Tensor> tiles, c10::optional<torch::Tensor> bounds, std::vector<double> poly, int64_t poly_at,
    int64_t ff, c10::optional<torch::Tensor> act, double eps) {
  const bool yf = f32_rows(y), cf = f32_rows(cache);
  TORCH_CHECK(y.dim() == 2 && y.is_contiguous() && y.size(1) % 8 == 0 && reinterpret_cast<uintptr_t>(y.data_ptr()) % 16 == 0);
  TORCH_CHECK(yf || !cf, "a 32-bit cache of 16-bit rows");
  const long t = y.size(0);
  const PagedRows b = paged_rows(pos, owner, tables, cache, t);
  TORCH_CHECK(heads >= 1 && kv_heads >= 1 && dk % 32 == 0 && dk >= dim && dim >= 1 && values >= 8 && values % 8 == 0);
  RowShape s{(int)(heads * dk), (int)(kv_heads * dk), (int)values, (int)dk, (int)(heads * dim), (int)(kv_heads * dim), 0, 1};
  const long columns = s.columns();
  TORCH_CHECK(y.size(1) >= columns && cache.size(2) == s.nk + s.nv && cache.size(2) % 8 == 0, "projection or cache too narrow");
  RowWeights w{opt(bias, columns), nullptr, opt(norm, s.nq + s.nk)};
  ConvState st{nullptr, nullptr, false};
  if (conv_w.has_value()) {
    TORCH_CHECK(conv_w->dim() == 2 && conv_w->size(0) >= 1 && conv_w->size(1) == columns);
    s.taps = conv_w->size(0);
    w.conv = opt(conv_w, s.taps * columns);
    if (s.taps > 1) {
      TORCH_CHECK(conv.has_value() && conv->dim() == 3 && conv->size(1) == s.taps && conv->size(2) == columns);
      TORCH_CHECK(slot.has_value() && slot->is_cuda() && slot->dtype() == torch::kInt32 && slot->is_contiguous());
      TORCH_CHECK(slot->numel() == tables.size(0) && conv->size(0) >= 1);
      s.slots = conv->size(0);
      st.inputs = const_cast<float*>(opt(conv, conv->numel()));
      st.slot = slot->data_ptr<int>();
      st.store = single;
      if (!single) {
        for (const auto& m : {tiles, bounds})
          TORCH_CHECK(m.has_value() && m->is_cuda() && m->dtype() == torch::kInt32 && m->is_contiguous());
        TORCH_CHECK(bounds->numel() == tables.size(0) + 1);
      }
    }
  }
  const Rotation r = rotation(quarters);
  TORCH_CHECK(r.turned <= dim, "rotation of ", r.turned, " of ", dim, " values");
  PolyPart pp{0, 0, 0, 0.f, 0.f, 0.f, 0.f};
  long act_stride = 0;
  if (!poly.empty()) {
    TORCH_CHECK(poly.size() == 4 && ff >= 1 && poly_at % 8 == 0 && act.has_value() && act->dtype() == y.dtype() && act->dim() == 2);
    pp = PolyPart{(int)poly_at, (int)ff, (int)act->size(1), (float)poly[0], (float)poly[1], (float)poly[2], (float)poly[3]};
    TORCH_CHECK(poly_at >= 0 && pp.padded >= ff && pp.padded % 8 == 0 && poly_at + pp.padded <= y.size(1));
    TORCH_CHECK(act->is_cuda() && act->dim() == 2 && act->stride(1) == 1 && act->size(0) == t);
    TORCH_CHECK(act->stride(0) % 8 == 0 && reinterpret_cast<uintptr_t>(act->data_ptr()) % 16 == 0);
    act_stride = act->stride(0);
  }
  auto q = torch::empty({t, (long)s.nq}, cache.options());
  if (t == 0) return q;
  const size_t lds = ((size_t)std::max(s.nq, s.nk) + r.turned) * 4;
  TORCH_CHECK(lds <= 160 * 1024 - 1024, "query projections of ", s.nq, " values are not supported");
  auto stream = at::cuda::getCurrentCUDAStream();
  const int half = r.turned / 2, most = std::max(s.nq, s.nk);
  if (!yf && t >= 512 && half % 8 == 0 && most <= 16 * 512 && s.taps <= 4 && s.taps != 1) {  // a prompt's rows
    const dim3 tiles_grid(((t + TILE_ROWS - 1) / TILE_ROWS + 7) / 8 * 8, 3);
    const size_t table = (size_t)TILE_ROWS * 2 * half * 4;
    TORCH_CHECK(table <= 32768, "rotation of ", r.turned, " values is not supported");
    const int threads = std::max(64, (most / 16 + 63) / 64 * 64);
#define PTN(TAPS, NT)                                                                                                   \
  prepare_tile_kernel<TAPS, NT><<<tiles_grid, threads, table, stream>>>(BF16P(y), (int)y.size(1), s, w, st, r,          \
                                                                        (float)turn_factor, b, BF16P(q), BF16P(cache),  \
                                                                        (float)eps, (int)t)
#define PT(TAPS)                        \
  do {                                  \
    if (threads <= 256) PTN(TAPS, 256); \
    else PTN(TAPS, 512);                \
  } while (0)
    switch (s.taps) {
      case 0: PT(0); break;
      case 2: PT(2); break;
      case 3: PT(3); break;
      default: PT(4);
    }
#undef PT
#undef PTN
    HIP_CHECK_LAST();
    if (!poly.empty()) {
      const auto poly_rows = &poly_kernel<unsigned short, 256>;
      poly_rows<<<dim3(t), 256, 0, stream>>>(BF16P(y), (int)y.size(1), (float)eps, pp, BF16P(*act), act_stride);
      HIP_CHECK_LAST();
    }
    conv_tail(y, s, w, st, single, pos, tiles, bounds);
    return q;
  }
  const bool spread = t >= 64;
  const dim3 grid(spread ? (t + 7) / 8 * 8 : t, poly.empty() ? 3 : 4);
#define PRN(TY, TC, NT)                                                                                                \
  do {                                                                                                                 \
    if (lds > 65536 - 1024) {                                                                                          \
      const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&prepare_rows_kernel<TY, TC, NT>),        \
                                               hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);                  \
      TORCH_CHECK(e == hipSuccess, "LDS request refused: ", hipGetErrorString(e));                                     \
    }                                                                                                                  \
    prepare_rows_kernel<TY, TC, NT><<<grid, NT, lds, stream>>>(                                                        \
        reinterpret_cast<const TY*>(y.data_ptr()), (int)y.size(1), s, w, st, r, (float)turn_factor, b,                 \
        reinterpret_cast<TC*>(q.data_ptr()), reinterpret_cast<TC*>(cache.data_ptr()), (float)eps, pp,                  \
        poly.empty() ? nullptr : reinterpret_cast<TY*>(act->data_ptr()), act_stride, (int)t, spread);                  \
  } while (0)
#define PR(TY, TC)                   \
  do {                               \
    if (t < 512) PRN(TY, TC, 1024);  \
    else PRN(TY, TC, 256);           \
  } while (0)
  if (cf) PR(float, float);
  else if (yf) PR(float, unsigned short);
  else PR(unsigned short, unsigned short);
#undef PR
#undef PRN
  HIP_CHECK_LAST();
  conv_tail(y, s, w, st, single, pos, tiles, bounds);
  return q;
}
