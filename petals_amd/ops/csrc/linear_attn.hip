// Gated linear attention for CDNA4 (gfx950): recurrent layers whose state is, per
// head, a matrix S [dim, vdim] in 32-bit with
//
//   S <- diag(g) S + k v^T;   o = S^T q
//
// in two forms:
//   forget gate  g per channel, f = l + (1 - l) sigmoid(z + b); k = 1 - f, q = silu(.)
//                (HGRN2), o normed per head
//   state space  g one number per head, exp(-a dt); k = dt B, q = C and v = x from a
//                short causal convolution with silu, B and C shared by groups of
//                heads; o + D x is gated and normed in groups (Mamba-2)
//
// A prompt is cut into chunks of 16 tokens. With G_i the product of the decays up to
// token i of its chunk and S0 the state before it,
//
//   QK_ij = sum_c q_i k_j G_i/G_j  (j <= i)
//   O     = (G q) S0 + QK V
//   S     = G_15 S0 + (G_15/G k)^T V
//
// Every ratio of decays is at most 1 and is taken as the exponential of a difference
// of logarithms, so nothing overflows however strong the decay.
//
//   forget_chunk_kernel  what does not depend on S, for all chunks at once
//   ssm_conv_kernel      the convolution of all rows
//   ssm_chunk_kernel     step sizes, decays and QK of all chunks
//   linear_scan_kernel   the chunks of a sequence in order, S in accumulators of
//                        32-bit MFMA products
//   ssm_conv_tail        the convolution's inputs that the next step needs
//   group_norm_kernel    gate and norm in groups
//   linear_decode_kernel one token per sequence, all of the above (of a state-space
//                        layer all but the norm) in one launch
//
// State: [slots, H, DK, DV] with DK, DV multiples of 16 (zeros past dim and vdim) and
// the convolution's inputs [slots, taps, channels], position p in row p % taps. A
// sequence whose first row stands at position 0 starts from zero whatever its slot
// holds.

#include "recurrence.h"
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>
#include <type_traits>

struct LinearShape {
  int heads, dim, vdim, dk, dv, slots;
};

// rows of a step in chunks, and the slots of their sequences
struct ChunkRows {
  const int* tiles;   // [n, 2] first row, row count
  const int* bounds;  // [S + 1] chunks of each sequence
  const int* pos;     // [T]
  const int* owner;   // [T]
  const int* slot;    // [S]
};

__device__ __forceinline__ float silu_f32(float x) { return x / (1.f + expf(-x)); }

// log2 of 1 - k for 0 <= k <= 1; near 0 by the series of log((1 - s)/(1 + s)) at
// s = k/(2 - k), which keeps the digits that 1 - k has lost
__device__ __forceinline__ float log2_of_rest(float k, float f) {
  if (k < 0.25f) {
    const float s = k / (2.f - k), t = s * s;
    float r = 1.f / 11.f;
    r = fmaf(r, t, 1.f / 9.f);
    r = fmaf(r, t, 1.f / 7.f);
    r = fmaf(r, t, 1.f / 5.f);
    r = fmaf(r, t, 1.f / 3.f);
    r = fmaf(r, t, 1.f);
    return -2.f * LOG2E * s * r;
  }
  return log2f(fmaxf(f, 1e-37f));
}

// f = lower + (1 - lower) sigmoid(z) and k = 1 - f, neither by cancellation
__device__ __forceinline__ void forget_gate(float z, float lower, float& f, float& k) {
  const float e = expf(-fabsf(z)), big = 1.f / (1.f + e), small = e * big;
  f = fmaf(1.f - lower, z > 0.f ? big : small, lower);
  k = (1.f - lower) * (z > 0.f ? small : big);
}

// ------------------------------------------------- forget gate: per chunk

// floats of one (chunk, head): G q [16][dk], G_15/G k [dk][16], QK [16][16], G_15 [dk]
__host__ __device__ __forceinline__ size_t forget_unit(int dk) { return (size_t)2 * CH * dk + CH * CH + dk; }

struct ForgetColumns {
  int q, f;  // first columns in the projection
};

// Grid: (chunks, heads), 256 threads: 16 per token. BY8: head size and columns are
// multiples of 8.
template <typename TY, bool BY8>
__global__ __launch_bounds__(256) void forget_chunk_kernel(
    const TY* __restrict__ y, int stride, ForgetColumns col, const float* __restrict__ bias,
    const float* __restrict__ lower, const int* __restrict__ tiles, LinearShape s, float* __restrict__ ws) {
  extern __shared__ float sm[];
  const int P = s.dk + 4;
  float* sq = sm;           // [16][P]
  float* sk = sq + CH * P;  // [16][P]
  float* sl = sk + CH * P;  // [16][P] log2 decays, then their running sums
  const int tid = threadIdx.x, i = tid >> 4, l16 = tid & 15;
  const int h = blockIdx.y;
  const int row0 = tiles[2 * blockIdx.x], n = tiles[2 * blockIdx.x + 1];
  const bool valid = i < n;
  const TY* yr = y + (size_t)(row0 + (valid ? i : 0)) * stride;
  float* w_qt = ws + ((size_t)blockIdx.x * s.heads + h) * forget_unit(s.dk);
  float* w_kh = w_qt + CH * s.dk;
  float* w_qk = w_kh + CH * s.dk;
  float* w_g = w_qk + CH * CH;

  if (BY8) {
    for (int c = l16 * 8; c < s.dk; c += 128) {
      float q[8], k[8], lg[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) q[e] = k[e] = lg[e] = 0.f;
      if (valid && c < s.dim) {
        const int at = h * s.dim + c;
        float z[8], b[8], lo[8];
        load8(yr + col.q + at, q);
        load8(yr + col.f + at, z);
        load8(bias + at, b);
        load8(lower + at, lo);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          float f;
          forget_gate(z[e] + b[e], lo[e], f, k[e]);
          lg[e] = log2_of_rest(k[e], f);
          q[e] = silu_f32(q[e]);
        }
      }
      store8(&sq[i * P + c], q);
      store8(&sk[i * P + c], k);
      store8(&sl[i * P + c], lg);
    }
  } else {
    for (int c = l16; c < s.dk; c += 16) {
      float q = 0.f, k = 0.f, lg = 0.f;
      if (valid && c < s.dim) {
        const int at = h * s.dim + c;
        float f;
        forget_gate(load_f32(yr + col.f + at) + bias[at], lower[at], f, k);
        lg = log2_of_rest(k, f);
        q = silu_f32(load_f32(yr + col.q + at));
      }
      sq[i * P + c] = q;
      sk[i * P + c] = k;
      sl[i * P + c] = lg;
    }
  }
  __syncthreads();
  for (int c = tid; c < s.dk; c += 256) {
    float sum = 0.f;
#pragma unroll
    for (int t = 0; t < CH; ++t) {
      sum += sl[t * P + c];
      sl[t * P + c] = sum;
    }
    w_g[c] = exp2f(sum);
  }
  __syncthreads();
  for (int c = l16; c < s.dk; c += 16) w_qt[i * s.dk + c] = sq[i * P + c] * exp2f(sl[i * P + c]);
  for (int idx = tid; idx < CH * s.dk; idx += 256) {
    const int c = idx >> 4, t = idx & 15;
    w_kh[idx] = sk[t * P + c] * exp2f(sl[15 * P + c] - sl[t * P + c]);
  }
  // pairs (i, j): 32-bit throughout
  const int j = l16;
  float qk = 0.f;
  if (j <= i) {
    for (int c = 0; c < s.dk; c += 4) {
      const f32x4 li = *reinterpret_cast<const f32x4*>(&sl[i * P + c]), lj = *reinterpret_cast<const f32x4*>(&sl[j * P + c]);
      const f32x4 qi = *reinterpret_cast<const f32x4*>(&sq[i * P + c]), kj = *reinterpret_cast<const f32x4*>(&sk[j * P + c]);
#pragma unroll
      for (int e = 0; e < 4; ++e) qk = fmaf(qi[e], kj[e] * exp2f(li[e] - lj[e]), qk);
    }
  }
  w_qk[i * CH + j] = qk;
}

// --------------------------------------- state space: convolution, per chunk

struct SsmShape {
  int heads, groups, dim, vdim, dk, taps, slots;
  int o_conv, o_dt;  // first columns of the convolution's inputs and of the step sizes in the projection
  __device__ __host__ int inner() const { return heads * vdim; }
  __device__ __host__ int channels() const { return inner() + 2 * groups * dim; }
  // columns of the convolved rows: x, then keys and queries, dk for each group
  __device__ __host__ int at_k() const { return (inner() + 7) / 8 * 8; }
  __device__ __host__ int at_q() const { return at_k() + groups * dk; }
  __device__ __host__ int mixed() const { return at_q() + groups * dk; }
};

struct ConvWeights {
  const float* w;     // [taps, channels]
  const float* bias;  // [channels]
};

// the channel of column c of the convolved rows, -1: padding
__device__ __forceinline__ int ssm_channel(const SsmShape& s, int c) {
  if (c < s.inner()) return c;
  if (c < s.at_k()) return -1;
  const int part = c >= s.at_q(), r = c - (part ? s.at_q() : s.at_k());
  const int g = r / s.dk, n = r - g * s.dk;
  return n < s.dim ? s.inner() + (part * s.groups + g) * s.dim + n : -1;
}

__device__ __forceinline__ void load_n(const float* p, float (&v)[1]) { v[0] = *p; }
__device__ __forceinline__ void load_n(const unsigned short* p, float (&v)[1]) { v[0] = bf16_to_f32(*p); }
template <typename T> __device__ __forceinline__ void load_n(const T* p, float (&v)[8]) { load8(p, v); }

#define CONV_ROWS 4  // rows of a thread

// 4 groups of CONV_ROWS rows x 64 groups of V columns per workgroup. V = 8 needs
// aligned groups; TAPS: the number of taps, 0 for any.
template <typename TY, int V, int TAPS>
__global__ __launch_bounds__(256) void ssm_conv_kernel(
    const TY* __restrict__ y, int stride, ConvWeights cw, const float* __restrict__ state, ChunkRows b, SsmShape s,
    int rows, float* __restrict__ mixed) {
  const int row0 = (blockIdx.x * 4 + threadIdx.x / 64) * CONV_ROWS, c = (blockIdx.y * 64 + (threadIdx.x & 63)) * V;
  if (row0 >= rows || c >= s.mixed()) return;
  const int ch = ssm_channel(s, c), n = min(CONV_ROWS, rows - row0);
  float* dst = mixed + (size_t)row0 * s.mixed() + c;
  const TY* src = y + (size_t)row0 * stride + s.o_conv + ch;
  const int first_seq = b.owner[row0];
  float acc[V], x[V], w[V], bias[V];
  if (ch < 0) {
    for (int r = 0; r < n; ++r)
#pragma unroll
      for (int e = 0; e < V; ++e) dst[(size_t)r * s.mixed() + e] = 0.f;
    return;
  }
  load_n(cw.bias + ch, bias);
  if constexpr (TAPS > 0) {
    // all inputs are rows of this step
    if (n == CONV_ROWS && b.owner[row0 + n - 1] == first_seq && row0 - b.tiles[2 * b.bounds[first_seq]] >= TAPS - 1) {
      float in[CONV_ROWS + TAPS - 1][V], taps[TAPS][V];
#pragma unroll
      for (int r = 0; r < CONV_ROWS + TAPS - 1; ++r) load_n(src + (long)(r - TAPS + 1) * stride, in[r]);
#pragma unroll
      for (int j = 0; j < TAPS; ++j) load_n(cw.w + (size_t)j * s.channels() + ch, taps[j]);
#pragma unroll
      for (int r = 0; r < CONV_ROWS; ++r) {
#pragma unroll
        for (int e = 0; e < V; ++e) {
          float sum = bias[e];
#pragma unroll
          for (int j = 0; j < TAPS; ++j) sum = fmaf(taps[j][e], in[r + j][e], sum);
          dst[(size_t)r * s.mixed() + e] = silu_f32(sum);
        }
      }
      return;
    }
  }
  for (int r = 0; r < n; ++r) {
    const int row = row0 + r, seq = b.owner[row], p = b.pos[row];
    const int back = row - b.tiles[2 * b.bounds[seq]];
    const int slot = min(max(b.slot[seq], 0), s.slots - 1);
#pragma unroll
    for (int e = 0; e < V; ++e) acc[e] = bias[e];
    for (int j = 0; j < s.taps; ++j) {
      const int ago = s.taps - 1 - j;
      if (ago <= back) load_n(src + (long)(r - ago) * stride, x);
      else if (p - ago >= 0) load_n(state + ((size_t)slot * s.taps + (p - ago) % s.taps) * s.channels() + ch, x);
      else continue;
      load_n(cw.w + (size_t)j * s.channels() + ch, w);
#pragma unroll
      for (int e = 0; e < V; ++e) acc[e] = fmaf(w[e], x[e], acc[e]);
    }
#pragma unroll
    for (int e = 0; e < V; ++e) dst[(size_t)r * s.mixed() + e] = silu_f32(acc[e]);
  }
}

// floats of one (chunk, head): QK [16][16], G [16], G_15/G dt [16]
#define SSM_UNIT (CH * CH + 2 * CH)

// Grid: (chunks, groups, batches of 16 heads of a group)
template <typename TY>
__global__ __launch_bounds__(256) void ssm_chunk_kernel(
    const TY* __restrict__ y, int stride, const float* __restrict__ mixed, const float* __restrict__ a_exp,
    const float* __restrict__ dt_bias, const int* __restrict__ tiles, SsmShape s, float* __restrict__ ws) {
  extern __shared__ float sm[];
  const int P = s.dk + 4;
  float* sk = sm;           // [16][P]
  float* sq = sk + CH * P;  // [16][P]
  __shared__ float s_dt[16][16], s_sum[16][16];
  const int tid = threadIdx.x, i = tid >> 4, j = tid & 15;
  const int g = blockIdx.y, per = s.heads / s.groups, h0 = blockIdx.z * 16, nh = min(16, per - h0);
  const int row0 = tiles[2 * blockIdx.x], n = tiles[2 * blockIdx.x + 1];
  for (int idx = tid; idx < CH * s.dk / 4; idx += 256) {
    const int t = idx / (s.dk / 4), c = (idx - t * (s.dk / 4)) * 4;
    const float* src = mixed + (size_t)(row0 + min(t, n - 1)) * s.mixed() + g * s.dk + c;
    *reinterpret_cast<f32x4*>(&sk[t * P + c]) = *reinterpret_cast<const f32x4*>(src + s.at_k());
    *reinterpret_cast<f32x4*>(&sq[t * P + c]) = *reinterpret_cast<const f32x4*>(src + s.at_q());
  }
  {  // head h0 + i, token j
    const int h = g * per + h0 + i;
    float dt = 0.f, sum = 0.f;
    if (i < nh && j < n) {
      dt = softplus_f32(load_f32(y + (size_t)(row0 + j) * stride + s.o_dt + h) + dt_bias[h]);
      sum = -a_exp[h] * dt * LOG2E;
    }
#pragma unroll
    for (int off = 1; off < 16; off <<= 1) {
      const float up = __shfl_up(sum, off, 16);
      if (j >= off) sum += up;
    }
    s_dt[i][j] = dt;
    s_sum[i][j] = sum;
  }
  __syncthreads();
  float base = 0.f;
  if (j <= i)
    for (int c = 0; c < s.dk; c += 4) {
      const f32x4 q = *reinterpret_cast<const f32x4*>(&sq[i * P + c]), k = *reinterpret_cast<const f32x4*>(&sk[j * P + c]);
#pragma unroll
      for (int e = 0; e < 4; ++e) base = fmaf(q[e], k[e], base);
    }
  float* unit = ws + ((size_t)blockIdx.x * s.heads + g * per + h0) * SSM_UNIT;
  for (int h = 0; h < nh; ++h)
    unit[(size_t)h * SSM_UNIT + tid] = j <= i ? base * exp2f(s_sum[h][i] - s_sum[h][j]) * s_dt[h][j] : 0.f;
  if (i < nh) {
    unit += (size_t)i * SSM_UNIT + CH * CH;
    unit[j] = exp2f(s_sum[i][j]);
    unit[CH + j] = exp2f(s_sum[i][15] - s_sum[i][j]) * s_dt[i][j];
  }
}

// Grid: (sequences, channels / 256)
template <typename TY>
__global__ __launch_bounds__(256) void ssm_conv_tail(
    const TY* __restrict__ y, int stride, ChunkRows b, float* __restrict__ conv, SsmShape s) {
  const int seq = blockIdx.x, ch = blockIdx.y * 256 + threadIdx.x;
  if (ch >= s.channels() || b.bounds[seq] >= b.bounds[seq + 1]) return;
  const int slot = min(max(b.slot[seq], 0), s.slots - 1);
  const int first = b.tiles[2 * b.bounds[seq]], last = b.bounds[seq + 1] - 1;
  const int end = b.tiles[2 * last] + b.tiles[2 * last + 1];
  for (int row = max(first, end - s.taps); row < end; ++row)
    conv[((size_t)slot * s.taps + b.pos[row] % s.taps) * s.channels() + ch] =
        load_f32(y + (size_t)row * stride + s.o_conv + ch);
}

// ------------------------------------------------------------------- scan

// what the scan reads beside a unit of the workspace per (chunk, head)
template <typename TV>
struct ScanInput {
  const float* ws;
  const TV* v;  // row stride v_stride, head h's values at column o_v + h * vdim
  int v_stride, o_v;
  // state space only
  const float* mixed;  // convolved rows
  int mixed_stride, at_k, at_q, per_group;
  const float* skip;   // [H] D
};  // mixed_stride is v_stride

template <int TPW, int NS, bool SSM>
struct ScanOperands {
  f32x4 q[TPW], k[TPW];     // A operands of the state's products
  f32x4 g[SSM ? 1 : TPW];   // decays of the chunk; SSM: the factors of k
  float g15, qg;            // SSM: the decay of the chunk, the factor of q
  float qk;                 // this wave's column of QK
  float v[NS][4];
};

// Grid: (heads, slices of 16 NS columns of S, sequences): the slices of a head, which
// share their operands, meet in one XCD's L2. The 4 waves hold the 16-row tiles of S
// in turn, TPW each, and each adds a quarter of QK V to its share of the result;
// operands are on their way 3 chunks ahead (1 if they are many).
template <typename TV, int TPW, int NS, bool SSM>
__global__ __launch_bounds__(256) void linear_scan_kernel(
    ScanInput<TV> in, ChunkRows b, float* __restrict__ state, float* __restrict__ out,  // [T, H * vdim]
    LinearShape s) {
  __shared__ float part[2][NS][4][4][WAVE];  // [buffer][slice][register][wave][lane]
  const int h = blockIdx.x, v0 = blockIdx.y * 16 * NS, seq = blockIdx.z;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE), lane = threadIdx.x & (WAVE - 1);
  const int col = lane & 15, hi = lane >> 4;
  const int c0 = b.bounds[seq], c1 = b.bounds[seq + 1];
  if (c0 >= c1) return;
  const int slot = min(max(b.slot[seq], 0), s.slots - 1);
  // a sequence's rows are consecutive and all its chunks but the last are full
  const int seq_row0 = b.tiles[2 * c0], rows = b.tiles[2 * c1 - 2] + b.tiles[2 * c1 - 1] - seq_row0;
  const bool fresh = b.pos[seq_row0] == 0;
  const int n_tiles = s.dk / 16;
  float* st = state + ((size_t)slot * s.heads + h) * s.dk * s.dv + v0 + col;
  f32x4 acc[NS][TPW];
#pragma unroll
  for (int u = 0; u < NS; ++u)
#pragma unroll
    for (int t = 0; t < TPW; ++t) {
      const int tile = wave + t * 4;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        acc[u][t][r] = !fresh && tile < n_tiles ? st[(size_t)(tile * 16 + hi * 4 + r) * s.dv + u * 16] : 0.f;
    }
  const float skip = SSM ? in.skip[h] : 0.f;
  // Addresses are a base that moves with the chunk plus offsets that do not. Rows past
  // the end of the last chunk read its last one.
  const int tail = rows - (c1 - 1 - c0) * CH - 1;
  unsigned row_v[4], tail_v[4], col_v[NS], at_row[TPW], at_col[TPW];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    row_v[r] = (hi * 4 + r) * in.v_stride;
    tail_v[r] = min(hi * 4 + r, tail) * in.v_stride;
  }
#pragma unroll
  for (int u = 0; u < NS; ++u) col_v[u] = min(u * 16 + col, s.vdim - 1 - v0);
#pragma unroll
  for (int t = 0; t < TPW; ++t) {
    const int tile = min(wave + t * 4, n_tiles - 1);
    at_row[t] = tile * 16 + hi * 4;
    at_col[t] = tile * 16 + col;
  }
  const unsigned row_q = col * in.mixed_stride, tail_q = min(col, tail) * in.mixed_stride;
  auto load = [&](int c, ScanOperands<TPW, NS, SSM>& o) {
    const size_t row0 = seq_row0 + (size_t)(c - c0) * CH;
    const bool last = c == c1 - 1;  // uniform
    if constexpr (SSM) {
      const float* unit = in.ws + ((size_t)c * s.heads + h) * SSM_UNIT;
      const float* key = in.mixed + row0 * in.mixed_stride + in.at_k + h / in.per_group * s.dk;
      const float* query = key + (in.at_q - in.at_k);
      o.qk = unit[(unsigned)(col * CH + hi * 4 + wave)];
      o.qg = unit[(unsigned)(CH * CH + col)];
      o.g15 = unit[CH * CH + 15];
      o.g[0] = *reinterpret_cast<const f32x4*>(unit + (unsigned)(CH * CH + CH + hi * 4));
      const unsigned rq = last ? tail_q : row_q;
#pragma unroll
      for (int t = 0; t < TPW; ++t) {
        o.q[t] = *reinterpret_cast<const f32x4*>(query + (rq + at_row[t]));
#pragma unroll
        for (int r = 0; r < 4; ++r) o.k[t][r] = key[(last ? tail_v[r] : row_v[r]) + at_col[t]];
      }
    } else {
      const float* unit = in.ws + ((size_t)c * s.heads + h) * forget_unit(s.dk);
      const float* kh = unit + CH * s.dk;
      const float* qk = kh + CH * s.dk;
      const float* g = qk + CH * CH;
      o.qk = qk[(unsigned)(col * CH + hi * 4 + wave)];
#pragma unroll
      for (int t = 0; t < TPW; ++t) {
        o.q[t] = *reinterpret_cast<const f32x4*>(unit + (unsigned)(col * s.dk + at_row[t]));
        o.k[t] = *reinterpret_cast<const f32x4*>(kh + (at_col[t] * CH + hi * 4));
        o.g[t] = *reinterpret_cast<const f32x4*>(g + at_row[t]);
      }
    }
    const TV* v = in.v + row0 * in.v_stride + in.o_v + h * s.vdim + v0;
#pragma unroll
    for (int u = 0; u < NS; ++u)
#pragma unroll
      for (int r = 0; r < 4; ++r) o.v[u][r] = load_f32(v + ((last ? tail_v[r] : row_v[r]) + col_v[u]));
  };
  float mine[NS] = {};  // this wave's row of each group of 4 rows of the last chunk's values
  // What the waves have left in LDS for chunk c. `between` runs when it is read, ahead
  // of the branch around the store.
  auto finish = [&](int c, auto&& between) {
    lds_barrier();
    float o[NS];
#pragma unroll
    for (int u = 0; u < NS; ++u) {
      const float(*share)[WAVE] = part[c & 1][u][wave];
      o[u] = (share[0][lane] + share[1][lane]) + (share[2][lane] + share[3][lane]);
      if (SSM) o[u] = fmaf(skip, mine[u], o[u]);
    }
    between();
    const int row = (c - c0) * CH + hi * 4 + wave;
    float* dst = out + ((seq_row0 + (long)(c - c0) * CH) * s.heads + h) * s.vdim + v0;
#pragma unroll
    for (int u = 0; u < NS; ++u)
      if (row >= 0 && row < rows && v0 + u * 16 + col < s.vdim)
        dst[(unsigned)((hi * 4 + wave) * s.heads * s.vdim + u * 16 + col)] = o[u];
  };
  // The products of chunk c, then the result of the one before: the waves do not wait
  // for each other's share of a chunk right after it.
  auto step = [&](int c, const ScanOperands<TPW, NS, SSM>& now) {
    f32x4 v[NS], q[TPW], k[TPW], p[NS][TPW], old[NS][TPW];
    float next[NS];
#pragma unroll
    for (int t = 0; t < TPW; ++t) {
      const bool live = wave + t * 4 < n_tiles;
      q[t] = now.q[t];
      k[t] = now.k[t];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (SSM) {
          q[t][r] *= now.qg;
          k[t][r] *= now.g[0][r];
        }
        // no branch around a product: the tile past the last one takes zeros
        k[t][r] = live ? k[t][r] : 0.f;
      }
    }
#pragma unroll
    for (int u = 0; u < NS; ++u) {
#pragma unroll
      for (int r = 0; r < 4; ++r) v[u][r] = v0 + u * 16 + col < s.vdim ? now.v[u][r] : 0.f;
      const float low = wave & 1 ? v[u][1] : v[u][0], high = wave & 1 ? v[u][3] : v[u][2];
      next[u] = wave & 2 ? high : low;
#pragma unroll
      for (int t = 0; t < TPW; ++t) {
        p[u][t] = f32x4{0.f, 0.f, 0.f, 0.f};
        old[u][t] = acc[u][t];
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[u][t][r] *= SSM ? now.g15 : now.g[SSM ? 0 : t][r];
      }
      p[u][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(now.qk, next[u], p[u][0], 0, 0, 0);
    }
    // independent chains side by side
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int t = 0; t < TPW; ++t)
#pragma unroll
        for (int u = 0; u < NS; ++u) {
          p[u][t] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[t][r], old[u][t][r], p[u][t], 0, 0, 0);
          acc[u][t] = __builtin_amdgcn_mfma_f32_16x16x4f32(k[t][r], v[u][r], acc[u][t], 0, 0, 0);
        }
    finish(c - 1, [&] {  // nothing is stored for the chunk before the first
#pragma unroll
      for (int u = 0; u < NS; ++u) {
        mine[u] = next[u];
#pragma unroll
        for (int t = 1; t < TPW; ++t) p[u][0] += p[u][t];
#pragma unroll
        for (int r = 0; r < 4; ++r) part[c & 1][u][r][wave][lane] = p[u][0][r];
      }
    });
  };
  auto load_ahead = [&](int c, ScanOperands<TPW, NS, SSM>& o) { load(min(c, c1 - 1), o); };
  ScanOperands<TPW, NS, SSM> o0, o1, o2, o3;  // written out: an indexed array would not stay in registers
  load_ahead(c0, o0);
  if constexpr (TPW <= 2) {
    load_ahead(c0 + 1, o1);
    load_ahead(c0 + 2, o2);
    int c = c0;
    for (; c + 4 <= c1; c += 4) {
      load_ahead(c + 3, o3);
      step(c, o0);
      load_ahead(c + 4, o0);
      step(c + 1, o1);
      load_ahead(c + 5, o1);
      step(c + 2, o2);
      load_ahead(c + 6, o2);
      step(c + 3, o3);
    }
    if (c < c1) step(c, o0);
    if (c + 1 < c1) step(c + 1, o1);
    if (c + 2 < c1) step(c + 2, o2);
  } else {
    int c = c0;
    for (; c + 2 <= c1; c += 2) {
      load_ahead(c + 1, o1);
      step(c, o0);
      load_ahead(c + 2, o0);
      step(c + 1, o1);
    }
    if (c < c1) step(c, o0);
  }
  finish(c1 - 1, [] {});
#pragma unroll
  for (int u = 0; u < NS; ++u)
#pragma unroll
    for (int t = 0; t < TPW; ++t) {
      const int tile = wave + t * 4;
      if (tile < n_tiles)
#pragma unroll
        for (int r = 0; r < 4; ++r) st[(size_t)(tile * 16 + hi * 4 + r) * s.dv + u * 16] = acc[u][t][r];
    }
}

// ------------------------------------------------------------------- norm

// out[t, g * size + c] = v / rms(v) * w over each of `groups` parts of a row, with
// v = o, or o * silu(gate). L threads per part. Grid: parts / (256 / L).
template <int L, typename TZ, typename TO>
__global__ __launch_bounds__(256) void group_norm_kernel(
    const float* __restrict__ o, const TZ* __restrict__ gate, long gate_stride, const float* __restrict__ w,
    int w_step, TO* __restrict__ out, int out_stride, int groups, int size, long total, bool by4, float eps) {
  extern __shared__ float rows[];
  __shared__ float red[4];
  const int tid = threadIdx.x, lane = tid % L;
  const long part = (long)blockIdx.x * (256 / L) + tid / L;
  float* v = rows + tid / L * size;
  const bool live = part < total;
  const long t = live ? part / groups : 0;
  const int g = live ? (int)(part - t * groups) : 0;
  const float* src = o + (t * groups + g) * size;
  const TZ* gs = gate ? gate + t * gate_stride + (long)g * size : nullptr;
  float ss = 0.f;
  if (live) {
    if (by4) {
      for (int c = lane * 4; c < size; c += L * 4) {
        f32x4 x = *reinterpret_cast<const f32x4*>(src + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          if (gs) x[e] *= silu_f32(load_f32(gs + c + e));
          ss = fmaf(x[e], x[e], ss);
        }
        *reinterpret_cast<f32x4*>(v + c) = x;
      }
    } else {
      for (int c = lane; c < size; c += L) {
        const float x = gs ? src[c] * silu_f32(load_f32(gs + c)) : src[c];
        v[c] = x;
        ss = fmaf(x, x, ss);
      }
    }
  }
#pragma unroll
  for (int off = (L < WAVE ? L : WAVE) / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, WAVE);
  if (L > WAVE) {
    if ((tid & (WAVE - 1)) == 0) red[tid / WAVE] = ss;
    __syncthreads();
    ss = (red[0] + red[1]) + (red[2] + red[3]);
  }
  if (!live) return;
  const float inv = 1.f / sqrtf(ss / size + eps);
  // each thread reads what it has written
  const float* ws = w + (long)g * w_step;
  TO* dst = out + t * out_stride + (long)g * size;
  if (by4) {
    for (int c = lane * 4; c < size; c += L * 4)
#pragma unroll
      for (int e = 0; e < 4; ++e) store_f32(dst + c + e, v[c + e] * inv * ws[c + e]);
  } else {
    for (int c = lane; c < size; c += L) store_f32(dst + c, v[c] * inv * ws[c]);
  }
}

// --------------------------------------------------------------- decoding

struct ForgetDecode {
  ForgetColumns col;
  int o_v;
  const float *bias, *lower, *norm;
  int out_stride;
  float eps;
};

struct SsmDecode {
  SsmShape s;
  ConvWeights cw;
  const float *a_exp, *dt_bias, *skip;
  float* conv;
};

// S is on its way while the vectors are made. Grid: (tokens, heads); row t is
// sequence t's only one. 512 threads hold S, 4 columns and NR rows each. D names the form.
template <typename TY, int NR, typename D>
__global__ __launch_bounds__(512) void linear_decode_kernel(
    const TY* __restrict__ y, int stride, D d, const int* __restrict__ pos, const int* __restrict__ slot_of,
    float* __restrict__ state, void* __restrict__ out, LinearShape s) {
  constexpr bool SSM = std::is_same<D, SsmDecode>::value;
  extern __shared__ float sm[];
  float* sq = sm;           // [dk]
  float* sk = sq + s.dk;    // [dk]
  float* sg = sk + s.dk;    // [dk] decays of a forget gate
  float* sv = sg + s.dk;    // [dv]
  float* red = sv + s.dv;   // [2048]
  const int tid = threadIdx.x, lane = tid & (WAVE - 1);
  const int row = blockIdx.x, h = blockIdx.y;
  const int p = pos[row], slot = min(max(slot_of[row], 0), s.slots - 1);
  const TY* yr = y + (size_t)row * stride;

  const int tpr = s.dv / 4, rpp = 512 / tpr;  // threads per row of S, rows per pass
  const int rg = tid / tpr, vc = (tid - rg * tpr) * 4;
  float* st = state + ((size_t)slot * s.heads + h) * s.dk * s.dv + vc;
  f32x4 acc[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int c = rg + i * rpp;
    acc[i] = p > 0 && rg < rpp && c < s.dk ? *reinterpret_cast<const f32x4*>(st + (size_t)c * s.dv)
                                           : f32x4{0.f, 0.f, 0.f, 0.f};
  }

  float decay = 0.f, dt = 1.f;
  if constexpr (SSM) {
    const SsmShape& m = d.s;
    dt = softplus_f32(load_f32(yr + m.o_dt + h) + d.dt_bias[h]);
    decay = exp2f(-d.a_exp[h] * dt * LOG2E);
    const int per = m.heads / m.groups, g = h / per, channels = m.channels(), ring_row = p % m.taps;
    const float* ring0 = d.conv + (size_t)slot * m.taps * channels;
#pragma unroll 1
    for (int i = tid; i < 2 * s.dk + s.dv; i += 512) {
      const int part = i < s.dk ? 0 : i < 2 * s.dk ? 1 : 2;  // queries, keys, values
      const int c = i - part * s.dk;
      float x = 0.f;
      if (c < (part < 2 ? s.dim : s.vdim)) {
        const int ch = part == 2 ? h * s.vdim + c : m.inner() + ((part == 0 ? m.groups : 0) + g) * s.dim + c;
        const float own = load_f32(yr + m.o_conv + ch);
        const float* w = d.cw.w + (size_t)(m.taps - 1) * channels + ch;
        const float* ring = ring0 + ch;
        x = fmaf(own, *w, d.cw.bias[ch]);
        for (int a0 = 1; a0 < m.taps; a0 += 4) {  // 4 loads on their way at once
          float v[4], wt[4];
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const int ago = a0 + e < m.taps ? a0 + e : 0;
            v[e] = ring[(size_t)(ring_row >= ago ? ring_row - ago : ring_row - ago + m.taps) * channels];
            wt[e] = w[-(long)ago * channels];
          }
#pragma unroll
          for (int e = 0; e < 4; ++e) x = a0 + e < m.taps && a0 + e <= p ? fmaf(wt[e], v[e], x) : x;
        }
        x = silu_f32(x);
        // this row of the ring is read by no other workgroup, and not used above
        if (part == 2 || h == g * per) d.conv[((size_t)slot * m.taps + ring_row) * channels + ch] = own;
      }
      (part == 0 ? sq : part == 1 ? sk : sv)[c] = x;
    }
  } else {
#pragma unroll 1
    for (int i = tid; i < s.dk + s.dv; i += 512) {
      if (i < s.dk) {
        float q = 0.f, f = 0.f, k = 0.f;
        if (i < s.dim) {
          const int at = h * s.dim + i;
          q = silu_f32(load_f32(yr + d.col.q + at));
          forget_gate(load_f32(yr + d.col.f + at) + d.bias[at], d.lower[at], f, k);
        }
        sq[i] = q;
        sk[i] = k;
        sg[i] = f;
      } else {
        const int c = i - s.dk;
        sv[c] = c < s.vdim ? load_f32(yr + d.o_v + h * s.vdim + c) : 0.f;
      }
    }
  }
  __syncthreads();
  if (rg < rpp) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(&sv[vc]);
    f32x4 sum = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int c = rg + i * rpp;
      if (c >= s.dk) break;
      const float g = SSM ? decay : sg[c], k = SSM ? sk[c] * dt : sk[c], q = sq[c];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        acc[i][e] = fmaf(k, v[e], g * acc[i][e]);
        sum[e] = fmaf(acc[i][e], q, sum[e]);
      }
      *reinterpret_cast<f32x4*>(st + (size_t)c * s.dv) = acc[i];
    }
    *reinterpret_cast<f32x4*>(&red[rg * s.dv + vc]) = sum;
  }
  __syncthreads();
  if constexpr (SSM) {
    for (int c = tid; c < s.vdim; c += 512) {
      float t = 0.f;
      for (int r = 0; r < rpp; ++r) t += red[r * s.dv + c];
      reinterpret_cast<float*>(out)[((size_t)row * s.heads + h) * s.vdim + c] = fmaf(d.skip[h], sv[c], t);
    }
  } else {
    __shared__ float wsum[8];
    float mine = 0.f;
    for (int c = tid; c < s.dv; c += 512) {
      float t = 0.f;
      for (int r = 0; r < rpp; ++r) t += red[r * s.dv + c];
      sv[c] = t;
      mine = fmaf(t, t, mine);
    }
    mine = wave_reduce_sum(mine);
    if (lane == 0) wsum[tid / WAVE] = mine;
    __syncthreads();
    float ss = 0.f;
#pragma unroll
    for (int w = 0; w < 8; ++w) ss += wsum[w];
    const float inv = 1.f / sqrtf(ss / s.vdim + d.eps);
    for (int c = tid; c < s.vdim; c += 512)
      store_f32(reinterpret_cast<TY*>(out) + (size_t)row * d.out_stride + h * s.vdim + c, sv[c] * inv * d.norm[c]);
  }
}

// ------------------------------------------------------------------- host

static int up16(int64_t n) { return (int)((n + 15) / 16 * 16); }

static bool aligned16(std::initializer_list<const torch::Tensor*> tensors) {
  for (const torch::Tensor* t : tensors)
    if (reinterpret_cast<uintptr_t>(t->data_ptr()) % 16 != 0) return false;
  return true;
}

static void allow_lds(const void* kernel, size_t lds) {
  if (lds <= 65536) return;
  const hipError_t e = hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  TORCH_CHECK(e == hipSuccess, "LDS request refused: ", hipGetErrorString(e));
}

static LinearShape linear_shape(const torch::Tensor& y, const torch::Tensor& state, int64_t heads, int64_t dim, int64_t vdim) {
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous());
  TORCH_CHECK(y.dtype() == torch::kFloat32 || y.dtype() == torch::kBFloat16);
  TORCH_CHECK(heads >= 1 && heads <= 65535 && dim >= 1 && vdim >= 1);
  LinearShape s;
  s.heads = heads, s.dim = dim, s.vdim = vdim, s.dk = up16(dim), s.dv = up16(vdim);
  TORCH_CHECK(state.dim() == 4 && state.size(1) == heads && state.size(2) == s.dk && state.size(3) == s.dv, "state");
  s.slots = state.size(0);
  check_f32(state, state.numel(), "state");
  return s;
}

static void check_columns(const torch::Tensor& y, int64_t first, int64_t n) {
  TORCH_CHECK(first >= 0 && first + n <= y.size(1), "columns ", first, " to ", first + n, " of ", y.size(1));
}

static ChunkRows chunk_rows(const torch::Tensor& tiles, const torch::Tensor& bounds, const torch::Tensor& pos,
                            const torch::Tensor& owner, const torch::Tensor& slot, long rows) {
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2);
  const long seqs = bounds.numel() - 1;
  TORCH_CHECK(seqs >= 1 && seqs <= 65535);
  check_i32(tiles, tiles.numel(), "chunks");
  check_i32(bounds, seqs + 1, "chunk bounds");
  check_i32(pos, rows, "positions");
  check_i32(owner, rows, "owners");
  check_i32(slot, seqs, "slots");
  return ChunkRows{tiles.data_ptr<int>(), bounds.data_ptr<int>(), pos.data_ptr<int>(), owner.data_ptr<int>(),
                   slot.data_ptr<int>()};
}

template <typename TV, bool SSM>
static void launch_scan(const ScanInput<TV>& in, const ChunkRows& b, long seqs, torch::Tensor& state, torch::Tensor& out,
                        const LinearShape& s) {
  TORCH_CHECK(s.dk <= 512, "key size ", s.dim, " is not supported");
  const int slices = s.dv / 16, tpw = (s.dk / 16 + 3) / 4;
  // two slices share their operands where there are workgroups enough without
  const bool two = slices % 2 == 0 && (long)s.heads * slices * seqs >= 512;
  const dim3 grid(s.heads, two ? slices / 2 : slices, seqs);
  auto stream = at::cuda::getCurrentCUDAStream();
#define LS2(T, N) \
  linear_scan_kernel<TV, T, N, SSM><<<grid, 256, 0, stream>>>(in, b, state.data_ptr<float>(), out.data_ptr<float>(), s)
#define LS(T)            \
  do {                   \
    if (two) LS2(T, 2);  \
    else LS2(T, 1);      \
  } while (0)
  if (tpw <= 1) LS(1);
  else if (tpw <= 2) LS(2);
  else if (tpw <= 4) LS(4);
  else LS(8);
#undef LS
#undef LS2
  HIP_CHECK_LAST();
}

// Rows of any number of sequences; returns o [T, H * vdim] 32-bit, not yet normed.
// cols: first columns of q, f and v in the projection y. Updates the state.
torch::Tensor forget_prefill(
    torch::Tensor y, torch::Tensor bias, torch::Tensor lower, torch::Tensor tiles, torch::Tensor bounds,
    torch::Tensor pos, torch::Tensor owner, torch::Tensor slot, torch::Tensor state, int64_t heads, int64_t dim,
    int64_t vdim, std::vector<int64_t> cols) {
  const LinearShape s = linear_shape(y, state, heads, dim, vdim);
  const long t = y.size(0), chunks = tiles.size(0), seqs = bounds.numel() - 1;
  TORCH_CHECK(cols.size() == 3);
  check_columns(y, cols[0], heads * dim);
  check_columns(y, cols[1], heads * dim);
  check_columns(y, cols[2], heads * vdim);
  check_f32(bias, heads * dim, "gate bias");
  check_f32(lower, heads * dim, "lower bounds");
  const ChunkRows b = chunk_rows(tiles, bounds, pos, owner, slot, t);
  TORCH_CHECK(s.dk <= 512, "key size ", dim, " is not supported");
  auto out = torch::empty({t, heads * vdim}, state.options());
  if (t == 0) return out;
  auto ws = torch::empty({(long)(chunks * heads * forget_unit(s.dk))}, state.options());
  auto stream = at::cuda::getCurrentCUDAStream();
  const size_t lds = (size_t)3 * CH * (s.dk + 4) * 4;
  const int stride = y.size(1);
  const ForgetColumns col{(int)cols[0], (int)cols[1]};
  const bool by8 = dim % 8 == 0 && stride % 8 == 0 && cols[0] % 8 == 0 && cols[1] % 8 == 0 && aligned16({&y, &bias, &lower});
#define FC(TY, BY8, YP)                                                                                                 \
  do {                                                                                                                  \
    allow_lds(reinterpret_cast<const void*>(&forget_chunk_kernel<TY, BY8>), lds);                                       \
    forget_chunk_kernel<TY, BY8><<<dim3(chunks, heads), 256, lds, stream>>>(YP, stride, col, bias.data_ptr<float>(),    \
                                                                            lower.data_ptr<float>(), b.tiles, s,        \
                                                                            ws.data_ptr<float>());                      \
    HIP_CHECK_LAST();                                                                                                   \
    launch_scan<TY, false>(ScanInput<TY>{ws.data_ptr<float>(), YP, stride, (int)cols[2], nullptr, 0, 0, 0, 1, nullptr}, \
                           b, seqs, state, out, s);                                                                     \
  } while (0)
  if (y.dtype() == torch::kFloat32) {
    if (by8) FC(float, true, y.data_ptr<float>());
    else FC(float, false, y.data_ptr<float>());
  } else {
    if (by8) FC(unsigned short, true, BF16P(y));
    else FC(unsigned short, false, BF16P(y));
  }
#undef FC
  return out;
}

static SsmShape ssm_shape(const torch::Tensor& y, const LinearShape& l, int64_t groups, int64_t o_conv, int64_t o_dt,
                          const torch::Tensor& conv_w, const torch::Tensor& conv_b, const torch::Tensor& a_exp,
                          const torch::Tensor& dt_bias, const torch::Tensor& skip, const torch::Tensor& conv) {
  TORCH_CHECK(groups >= 1 && l.heads % groups == 0);
  SsmShape s;
  s.heads = l.heads, s.groups = groups, s.dim = l.dim, s.vdim = l.vdim, s.dk = l.dk, s.slots = l.slots;
  s.o_conv = o_conv, s.o_dt = o_dt;
  TORCH_CHECK(conv_w.dim() == 2 && conv_w.size(0) >= 1);
  s.taps = conv_w.size(0);
  check_columns(y, o_conv, s.channels());
  check_columns(y, o_dt, s.heads);
  check_f32(conv_w, (long)s.taps * s.channels(), "convolution weights");
  check_f32(conv_b, s.channels(), "convolution bias");
  check_f32(a_exp, s.heads, "decay rates");
  check_f32(dt_bias, s.heads, "step bias");
  check_f32(skip, s.heads, "skip");
  TORCH_CHECK(conv.dim() == 3 && conv.size(0) == s.slots && conv.size(1) == s.taps && conv.size(2) == s.channels(), "conv state");
  check_f32(conv, conv.numel(), "conv state");
  return s;
}

// Rows of any number of sequences; returns o + D x [T, H * vdim] 32-bit, not yet
// gated. o_conv, o_dt: first columns of the convolution's inputs (x, keys, queries)
// and of the step sizes in the projection y. Updates both states.
torch::Tensor ssm_prefill(
    torch::Tensor y, torch::Tensor conv_w, torch::Tensor conv_b, torch::Tensor a_exp, torch::Tensor dt_bias,
    torch::Tensor skip, torch::Tensor tiles, torch::Tensor bounds, torch::Tensor pos, torch::Tensor owner,
    torch::Tensor slot, torch::Tensor state, torch::Tensor conv, int64_t heads, int64_t groups, int64_t dim,
    int64_t vdim, int64_t o_conv, int64_t o_dt) {
  const LinearShape l = linear_shape(y, state, heads, dim, vdim);
  const SsmShape s = ssm_shape(y, l, groups, o_conv, o_dt, conv_w, conv_b, a_exp, dt_bias, skip, conv);
  const long t = y.size(0), chunks = tiles.size(0), seqs = bounds.numel() - 1;
  const ChunkRows b = chunk_rows(tiles, bounds, pos, owner, slot, t);
  TORCH_CHECK(s.dk <= 512 && groups <= 65535, "state size ", dim, " is not supported");
  auto out = torch::empty({t, heads * vdim}, state.options());
  if (t == 0) return out;
  auto ws = torch::empty({(long)(chunks * heads * SSM_UNIT)}, state.options());
  auto mixed = torch::empty({t, s.mixed()}, state.options());
  auto stream = at::cuda::getCurrentCUDAStream();
  const int stride = y.size(1), per = s.heads / s.groups;
  const bool by8 = s.inner() % 8 == 0 && dim % 8 == 0 && stride % 8 == 0 && o_conv % 8 == 0 && s.channels() % 8 == 0 &&
                   aligned16({&y, &conv_w, &conv_b, &conv});
  const size_t lds = (size_t)2 * CH * (s.dk + 4) * 4;
  const ConvWeights cw{conv_w.data_ptr<float>(), conv_b.data_ptr<float>()};
  const dim3 chunk_grid(chunks, groups, (per + 15) / 16);
#define SC(TY, YP, V, TAPS)                                                                                         \
  ssm_conv_kernel<TY, V, TAPS><<<dim3((t + 4 * CONV_ROWS - 1) / (4 * CONV_ROWS), (s.mixed() + 64 * V - 1) / (64 * V)), \
                                 256, 0, stream>>>(YP, stride, cw, conv.data_ptr<float>(), b, s, (int)t,            \
                                                   mixed.data_ptr<float>())
#define SP(TY, YP)                                                                                                  \
  do {                                                                                                              \
    if (by8 && s.taps == 4) SC(TY, YP, 8, 4);                                                                       \
    else if (by8) SC(TY, YP, 8, 0);                                                                                 \
    else SC(TY, YP, 1, 0);                                                                                          \
    HIP_CHECK_LAST();                                                                                               \
    ssm_conv_tail<TY><<<dim3(seqs, (s.channels() + 255) / 256), 256, 0, stream>>>(YP, stride, b,                    \
                                                                                  conv.data_ptr<float>(), s);       \
    HIP_CHECK_LAST();                                                                                               \
    allow_lds(reinterpret_cast<const void*>(&ssm_chunk_kernel<TY>), lds + 2048);                                    \
    ssm_chunk_kernel<TY><<<chunk_grid, 256, lds, stream>>>(YP, stride, mixed.data_ptr<float>(),                     \
                                                           a_exp.data_ptr<float>(), dt_bias.data_ptr<float>(),      \
                                                           b.tiles, s, ws.data_ptr<float>());                       \
    HIP_CHECK_LAST();                                                                                               \
  } while (0)
  if (y.dtype() == torch::kFloat32) SP(float, y.data_ptr<float>());
  else SP(unsigned short, BF16P(y));
#undef SP
#undef SC
  launch_scan<float, true>(
      ScanInput<float>{ws.data_ptr<float>(), mixed.data_ptr<float>(), s.mixed(), 0, mixed.data_ptr<float>(), s.mixed(),
                       s.at_k(), s.at_q(), per, skip.data_ptr<float>()},
      b, seqs, state, out, l);
  return out;
}

// o [T, n] 32-bit in `groups` equal parts; gate [T, n] view or absent; w [n], or one
// part's that all share. Returns [T, width], zero past n.
torch::Tensor group_norm(torch::Tensor o, c10::optional<torch::Tensor> gate, torch::Tensor w, int64_t groups,
                         int64_t width, bool f32, double eps) {
  TORCH_CHECK(o.dim() == 2 && groups >= 1 && o.size(1) % groups == 0);
  const long t = o.size(0), n = o.size(1), size = n / groups, total = t * groups;
  check_f32(o, t * n, "rows");
  TORCH_CHECK(w.numel() == n || w.numel() == size);
  check_f32(w, w.numel(), "norm weights");
  TORCH_CHECK(width >= n);
  bool zf = true, by4 = size % 4 == 0;
  const void* zp = nullptr;
  long zs = 0;
  if (gate.has_value()) {
    zf = gate->dtype() == torch::kFloat32;
    TORCH_CHECK(gate->is_cuda() && (zf || gate->dtype() == torch::kBFloat16) && gate->dim() == 2 && gate->stride(1) == 1 &&
                gate->size(0) == t && gate->size(1) == n);
    zp = gate->data_ptr();
    zs = gate->stride(0);
  }
  const auto opt = o.options().dtype(f32 ? torch::kFloat32 : torch::kBFloat16);
  auto out = width == n ? torch::empty({t, width}, opt) : torch::zeros({t, width}, opt);
  if (t == 0) return out;
  by4 = by4 && aligned16({&o});
  const int lanes = size <= 128 ? 16 : size <= 512 ? 64 : 256;
  const size_t lds = (size_t)(256 / lanes) * size * 4;
  TORCH_CHECK(lds <= 150000, "groups of ", size, " values are not supported");
  const long blocks = (total + 256 / lanes - 1) / (256 / lanes);
  const int w_step = w.numel() == size ? 0 : (int)size;
  auto stream = at::cuda::getCurrentCUDAStream();
#define GN2(L, TZ, TO)                                                                                             \
  do {                                                                                                             \
    allow_lds(reinterpret_cast<const void*>(&group_norm_kernel<L, TZ, TO>), lds + 64);                             \
    group_norm_kernel<L, TZ, TO><<<blocks, 256, lds, stream>>>(                                                    \
        o.data_ptr<float>(), reinterpret_cast<const TZ*>(zp), zs, w.data_ptr<float>(), w_step,                     \
        reinterpret_cast<TO*>(out.data_ptr()), (int)width, (int)groups, (int)size, total, by4, (float)eps);        \
  } while (0)
#define GN(TZ, TO)                          \
  do {                                      \
    if (lanes == 16) GN2(16, TZ, TO);       \
    else if (lanes == 64) GN2(64, TZ, TO);  \
    else GN2(256, TZ, TO);                  \
  } while (0)
  if (zf && f32) GN(float, float);
  else if (zf) GN(float, unsigned short);
  else if (f32) GN(unsigned short, float);
  else GN(unsigned short, unsigned short);
#undef GN
#undef GN2
  HIP_CHECK_LAST();
  return out;
}

static size_t decode_lds(const LinearShape& s) { return (size_t)(3 * s.dk + s.dv + 2048) * 4; }

// rows of S per thread in the decoding kernel, 0 if it does not take these sizes
static int decode_rows(const LinearShape& s) {
  if (s.dv > 2048 || decode_lds(s) > 60000) return 0;
  const int rpp = 512 / (s.dv / 4), need = (s.dk + rpp - 1) / rpp;
  return need <= 4 ? 4 : need <= 8 ? 8 : need <= 16 ? 16 : need <= 32 ? 32 : 0;
}

bool linear_decodes(int64_t dim, int64_t vdim) {
  LinearShape s;
  s.dk = up16(dim), s.dv = up16(vdim);
  return decode_rows(s) > 0;
}

template <typename TY, typename D>
static void launch_decode(const TY* y, int stride, long t, const D& d, const torch::Tensor& pos, const torch::Tensor& slot,
                          torch::Tensor& state, void* out, const LinearShape& s) {
  check_i32(pos, t, "positions");
  TORCH_CHECK(slot.numel() == t, "one row per sequence");
  check_i32(slot, t, "slots");
  const int nr = decode_rows(s);
  TORCH_CHECK(nr > 0, "head sizes ", s.dim, " and ", s.vdim, " are not supported");
  if (t == 0) return;
  auto stream = at::cuda::getCurrentCUDAStream();
#define LD(N)                                                                                         \
  linear_decode_kernel<TY, N, D><<<dim3(t, s.heads), 512, decode_lds(s), stream>>>(                   \
      y, stride, d, pos.data_ptr<int>(), slot.data_ptr<int>(), state.data_ptr<float>(), out, s)
  if (nr == 4) LD(4);
  else if (nr == 8) LD(8);
  else if (nr == 16) LD(16);
  else LD(32);
#undef LD
  HIP_CHECK_LAST();
}

// One row per sequence; returns [T, width] in y's dtype, normed per head.
torch::Tensor forget_decode(
    torch::Tensor y, torch::Tensor bias, torch::Tensor lower, torch::Tensor norm_w, torch::Tensor pos,
    torch::Tensor slot, torch::Tensor state, int64_t heads, int64_t dim, int64_t vdim, std::vector<int64_t> cols,
    int64_t width, double eps) {
  const LinearShape s = linear_shape(y, state, heads, dim, vdim);
  TORCH_CHECK(cols.size() == 3 && width >= heads * vdim);
  check_columns(y, cols[0], heads * dim);
  check_columns(y, cols[1], heads * dim);
  check_columns(y, cols[2], heads * vdim);
  check_f32(bias, heads * dim, "gate bias");
  check_f32(lower, heads * dim, "lower bounds");
  check_f32(norm_w, vdim, "norm weights");
  const long t = y.size(0);
  auto out = width == heads * vdim ? torch::empty({t, width}, y.options()) : torch::zeros({t, width}, y.options());
  const ForgetDecode d{{(int)cols[0], (int)cols[1]}, (int)cols[2], bias.data_ptr<float>(), lower.data_ptr<float>(),
                       norm_w.data_ptr<float>(), (int)width, (float)eps};
  if (y.dtype() == torch::kFloat32)
    launch_decode<float>(y.data_ptr<float>(), (int)y.size(1), t, d, pos, slot, state, out.data_ptr(), s);
  else
    launch_decode<unsigned short>(BF16P(y), (int)y.size(1), t, d, pos, slot, state, out.data_ptr(), s);
  return out;
}

// One row per sequence; returns o + D x [T, H * vdim] 32-bit, not yet gated.
torch::Tensor ssm_decode(
    torch::Tensor y, torch::Tensor conv_w, torch::Tensor conv_b, torch::Tensor a_exp, torch::Tensor dt_bias,
    torch::Tensor skip, torch::Tensor pos, torch::Tensor slot, torch::Tensor state, torch::Tensor conv, int64_t heads,
    int64_t groups, int64_t dim, int64_t vdim, int64_t o_conv, int64_t o_dt) {
  const LinearShape l = linear_shape(y, state, heads, dim, vdim);
  SsmDecode d;
  d.s = ssm_shape(y, l, groups, o_conv, o_dt, conv_w, conv_b, a_exp, dt_bias, skip, conv);
  d.cw = ConvWeights{conv_w.data_ptr<float>(), conv_b.data_ptr<float>()};
  d.a_exp = a_exp.data_ptr<float>(), d.dt_bias = dt_bias.data_ptr<float>(), d.skip = skip.data_ptr<float>();
  d.conv = conv.data_ptr<float>();
  const long t = y.size(0);
  auto out = torch::empty({t, heads * vdim}, state.options());
  if (y.dtype() == torch::kFloat32)
    launch_decode<float>(y.data_ptr<float>(), (int)y.size(1), t, d, pos, slot, state, out.data_ptr(), l);
  else
    launch_decode<unsigned short>(BF16P(y), (int)y.size(1), t, d, pos, slot, state, out.data_ptr(), l);
  return out;
}
