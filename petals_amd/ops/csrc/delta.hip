// Gated delta rule with a decay per key channel for CDNA4 (gfx950). Per head, S
// [dim, vdim] in 32-bit:
//
//   S <- g * S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
//
// with q, k, v from short causal convolutions (silu), q and k made unit vectors,
// g = exp(-exp(A) softplus(a + dt_bias)) and o normed and gated at the end.
//
// A prompt is cut into chunks of 16 tokens. With G_i the product of the decays
// up to token i of its chunk and S0 the state before it,
//
//   A_ij  = sum_c k_i k_j G_i/G_j  (j < i)      QK_ij = sum_c q_i k_j G_i/G_j  (j <= i)
//   U     = (I + beta A)^-1 beta (V - (G k) S0)
//   O     = (G q) S0 + QK U
//   S     = G_15 S0 + (G_15/G k)^T U
//
// Every ratio of decays is at most 1 and is taken as the exponential of a
// difference of logarithms, so nothing overflows however strong the decay.
//
//   delta_chunk_kernel   what does not depend on S, for all chunks at once
//   delta_scan_kernel    the chunks of a sequence in order, S in accumulators of
//                        32-bit MFMA products (16 columns of S per workgroup)
//   delta_conv_tail      the convolution's inputs that the next step needs
//   delta_norm_kernel    norm and gate of the result
//   delta_decode_kernel  one token per sequence, all of the above in one launch
//
// State: delta [slots, H, DK, DV] with DK, DV multiples of 16 (zeros past dim and
// vdim) and conv [slots, taps, channels], position p in row p % taps. A sequence
// whose first row stands at position 0 starts from zero whatever its slot holds.

#include "recurrence.h"
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>

struct DeltaShape {
  int heads, kv_heads, dim, vdim, dk, dv, taps, slots;
  int oq, ok, ov, ob;  // first columns of queries, keys, values and beta in the projection
  __device__ __host__ int channels() const { return 2 * kv_heads * dim + heads * vdim; }
};

// raw convolution inputs: rows of this step, before them the state
template <typename TY>
struct ConvInput {
  const TY* y;  // [T, stride]
  int stride;
  const float* w;      // [taps, channels]
  const float* state;  // [slots, taps, channels]
};

// silu of the convolution at row `row`, which is the i-th of this step's rows of
// its sequence (or of the part of it that `back` rows lead up to)
template <typename TY>
__device__ __forceinline__ float conv_silu(
    const ConvInput<TY>& in, const DeltaShape& s, int row, int back, int pos, int slot, int col, int ch) {
  float acc = 0.f;
  for (int j = 0; j < s.taps; ++j) {
    const int ago = s.taps - 1 - j;
    float x = 0.f;
    if (ago <= back) x = load_f32(in.y + (size_t)(row - ago) * in.stride + col);
    else if (pos - ago >= 0) x = in.state[((size_t)slot * s.taps + (pos - ago) % s.taps) * s.channels() + ch];
    acc = fmaf(in.w[j * s.channels() + ch], x, acc);
  }
  return acc / (1.f + expf(-acc));
}

// 8 neighbouring channels at once (aligned groups)
template <typename TY>
__device__ __forceinline__ void conv_silu8(
    const ConvInput<TY>& in, const DeltaShape& s, int row, int back, int pos, int slot, int col, int ch, float* out) {
  float acc[8], x[8], w[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) acc[e] = 0.f;
  for (int j = 0; j < s.taps; ++j) {
    const int ago = s.taps - 1 - j;
    if (ago <= back) load8(in.y + (size_t)(row - ago) * in.stride + col, x);
    else if (pos - ago >= 0) load8(in.state + ((size_t)slot * s.taps + (pos - ago) % s.taps) * s.channels() + ch, x);
    else continue;
    load8(in.w + (size_t)j * s.channels() + ch, w);
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[e] = fmaf(w[e], x[e], acc[e]);
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) out[e] = acc[e] / (1.f + expf(-acc[e]));
}

// log2 of the decay
__device__ __forceinline__ float log_decay(float a, float dt_bias, float a_exp) {
  return -a_exp * softplus_f32(a + dt_bias) * LOG2E;
}

// floats of one (chunk, head) in the workspace
__host__ __device__ __forceinline__ size_t unit_size(int dk, int dv) {
  return (size_t)3 * CH * dk + CH * dv + 2 * CH * CH + dk;
}

// ---------------------------------------------------------------- per chunk

// Grid: (chunks, heads), 256 threads: 16 per token. BY8: head sizes and columns
// are multiples of 8.
template <typename TY, bool BY8>
__global__ __launch_bounds__(256) void delta_chunk_kernel(
    ConvInput<TY> in, const float* __restrict__ a,  // a: [T, H * dim]
    const float* __restrict__ a_exp, const float* __restrict__ dt_bias, const int* __restrict__ tiles,
    const int* __restrict__ bounds, const int* __restrict__ pos, const int* __restrict__ owner,
    const int* __restrict__ slot_of, DeltaShape s, float* __restrict__ ws) {
  extern __shared__ float sm[];
  const int P = s.dk + 4;
  float* sq = sm;            // [16][P]
  float* sk = sq + CH * P;   // [16][P]
  float* sl = sk + CH * P;   // [16][P] log2 decays, then their running sums
  float* sa = sl + CH * P;   // [16][17]
  float* sb = sa + CH * 17;  // [16] beta
  const int tid = threadIdx.x, i = tid >> 4, l16 = tid & 15;
  const int h = blockIdx.y, kvh = h / (s.heads / s.kv_heads);
  const int row0 = tiles[2 * blockIdx.x], n = tiles[2 * blockIdx.x + 1];
  const int seq = owner[row0];
  const int slot = min(max(slot_of[seq], 0), s.slots - 1);
  const int seq_row0 = tiles[2 * bounds[seq]];
  const bool valid = i < n;
  const int row = row0 + (valid ? i : 0), back = row - seq_row0, p = pos[row];
  float* unit = ws + ((size_t)blockIdx.x * s.heads + h) * unit_size(s.dk, s.dv);
  float* w_kt = unit;                     // [16][dk]  G k
  float* w_qt = w_kt + CH * s.dk;         // [16][dk]  G q
  float* w_kh = w_qt + CH * s.dk;         // [dk][16]  G_15/G k, transposed
  float* w_v = w_kh + CH * s.dk;          // [16][dv]
  float* w_t = w_v + CH * s.dv;           // [16][16]  (I + beta A)^-1 beta
  float* w_qk = w_t + CH * CH;            // [16][16]
  float* w_g = w_qk + CH * CH;            // [dk]      G_15

  float q2 = 0.f, k2 = 0.f;
  if (BY8) {
    for (int c = l16 * 8; c < s.dk; c += 128) {
      float q[8], k[8], lg[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) q[e] = k[e] = lg[e] = 0.f;
      if (valid && c < s.dim) {
        const int cq = kvh * s.dim + c, ca = h * s.dim + c;
        conv_silu8(in, s, row, back, p, slot, s.oq + cq, cq, q);
        conv_silu8(in, s, row, back, p, slot, s.ok + cq, s.kv_heads * s.dim + cq, k);
        float b[8];
        load8(a + (size_t)row * s.heads * s.dim + ca, lg);
        load8(dt_bias + ca, b);
#pragma unroll
        for (int e = 0; e < 8; ++e) lg[e] = log_decay(lg[e], b[e], a_exp[h]);
      }
      store8(&sq[i * P + c], q);
      store8(&sk[i * P + c], k);
      store8(&sl[i * P + c], lg);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        q2 = fmaf(q[e], q[e], q2);
        k2 = fmaf(k[e], k[e], k2);
      }
    }
    for (int c = l16 * 8; c < s.dv; c += 128) {
      float v[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = 0.f;
      const int cv = h * s.vdim + c;
      if (valid && c < s.vdim) conv_silu8(in, s, row, back, p, slot, s.ov + cv, 2 * s.kv_heads * s.dim + cv, v);
      store8(w_v + i * s.dv + c, v);
    }
  }
  for (int c = BY8 ? s.dk : l16; c < s.dk; c += 16) {
    float q = 0.f, k = 0.f, lg = 0.f;
    if (valid && c < s.dim) {
      const int cq = kvh * s.dim + c;
      q = conv_silu(in, s, row, back, p, slot, s.oq + cq, cq);
      k = conv_silu(in, s, row, back, p, slot, s.ok + cq, s.kv_heads * s.dim + cq);
      const int ca = h * s.dim + c;
      lg = log_decay(a[(size_t)row * s.heads * s.dim + ca], dt_bias[ca], a_exp[h]);
    }
    sq[i * P + c] = q;
    sk[i * P + c] = k;
    sl[i * P + c] = lg;
    q2 = fmaf(q, q, q2);
    k2 = fmaf(k, k, k2);
  }
  const float qn = 1.f / sqrtf(group16_reduce_sum(q2) + 1e-6f) / sqrtf((float)s.dim);
  const float kn = 1.f / sqrtf(group16_reduce_sum(k2) + 1e-6f);
  __syncthreads();  // a row's channels were written by other lanes
  for (int c = l16; c < s.dk; c += 16) {
    sq[i * P + c] *= qn;
    sk[i * P + c] *= kn;
  }
  for (int c = BY8 ? s.dv : l16; c < s.dv; c += 16) {
    float v = 0.f;
    if (valid && c < s.vdim) {
      const int cv = h * s.vdim + c;
      v = conv_silu(in, s, row, back, p, slot, s.ov + cv, 2 * s.kv_heads * s.dim + cv);
    }
    w_v[i * s.dv + c] = v;
  }
  if (l16 == 0) sb[i] = valid ? 1.f / (1.f + expf(-load_f32(in.y + (size_t)row * in.stride + s.ob + h))) : 0.f;
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
  for (int c = l16; c < s.dk; c += 16) {
    const float e = exp2f(sl[i * P + c]);
    w_kt[i * s.dk + c] = sk[i * P + c] * e;
    w_qt[i * s.dk + c] = sq[i * P + c] * e;
  }
  for (int idx = tid; idx < CH * s.dk; idx += 256) {
    const int c = idx >> 4, t = idx & 15;
    w_kh[idx] = sk[t * P + c] * exp2f(sl[15 * P + c] - sl[t * P + c]);
  }
  // pairs (i, j): 32-bit throughout
  const int j = l16;
  float kk = 0.f, qk = 0.f;
  if (j <= i) {
    for (int c = 0; c < s.dk; c += 4) {
      const f32x4 li = *reinterpret_cast<const f32x4*>(&sl[i * P + c]), lj = *reinterpret_cast<const f32x4*>(&sl[j * P + c]);
      const f32x4 ki = *reinterpret_cast<const f32x4*>(&sk[i * P + c]), kj = *reinterpret_cast<const f32x4*>(&sk[j * P + c]);
      const f32x4 qi = *reinterpret_cast<const f32x4*>(&sq[i * P + c]);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float kr = kj[e] * exp2f(li[e] - lj[e]);
        kk = fmaf(ki[e], kr, kk);
        qk = fmaf(qi[e], kr, qk);
      }
    }
  }
  sa[i * 17 + j] = j < i ? kk : 0.f;
  w_qk[i * CH + j] = j <= i ? qk : 0.f;
  __syncthreads();
  if (tid < CH) {  // column tid of the inverse, by forward substitution
    float t[CH];
#pragma unroll
    for (int r = 0; r < CH; ++r) {
      float sum = 0.f;
#pragma unroll
      for (int c = 0; c < r; ++c) sum = fmaf(sa[r * 17 + c], t[c], sum);
      t[r] = (r == tid ? 1.f : 0.f) - sb[r] * sum;
      w_t[r * CH + tid] = t[r] * sb[tid];
    }
  }
}

// ------------------------------------------------------------------- scan

template <int TPW>
struct ChunkOperands {
  f32x4 kt[TPW], qt[TPW], kh[TPW], g[TPW], t, qk;
  float v[4];
};

// Grid: (heads, 16-column slices of S, sequences): the slices of a head, which
// share their operands, meet in one XCD's L2. The 4 waves hold the 16-row tiles
// of S in turn, TPW each; operands are on their way 3 chunks ahead (1 if they are many).
template <int TPW>
__global__ __launch_bounds__(256) void delta_scan_kernel(
    const float* __restrict__ ws, const int* __restrict__ tiles, const int* __restrict__ bounds,
    const int* __restrict__ pos, const int* __restrict__ slot_of, float* __restrict__ state,
    float* __restrict__ out,  // [T, H, vdim]
    DeltaShape s) {
  __shared__ f32x4 part[2][4][2][WAVE];
  const int h = blockIdx.x, v0 = blockIdx.y * 16, seq = blockIdx.z;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE), lane = threadIdx.x & (WAVE - 1);
  const int col = lane & 15, hi = lane >> 4;
  const int c0 = bounds[seq], c1 = bounds[seq + 1];
  if (c0 >= c1) return;
  const int slot = min(max(slot_of[seq], 0), s.slots - 1);
  const bool fresh = pos[tiles[2 * c0]] == 0;
  const int n_tiles = s.dk / 16;
  float* st = state + ((size_t)slot * s.heads + h) * s.dk * s.dv + v0 + col;
  f32x4 acc[TPW];
#pragma unroll
  for (int t = 0; t < TPW; ++t) {
    const int tile = wave + t * 4;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      acc[t][r] = !fresh && tile < n_tiles ? st[(size_t)(tile * 16 + hi * 4 + r) * s.dv] : 0.f;
  }
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  auto load = [&](int c, ChunkOperands<TPW>& o) {
    const float* unit = ws + ((size_t)c * s.heads + h) * unit_size(s.dk, s.dv);
    const float* kh = unit + 2 * CH * s.dk;
    const float* v = kh + CH * s.dk;
    const float* tt = v + CH * s.dv;
    const float* g = tt + 2 * CH * CH;
#pragma unroll
    for (int t = 0; t < TPW; ++t) {
      const int tile = min(wave + t * 4, n_tiles - 1);
      o.kt[t] = *reinterpret_cast<const f32x4*>(unit + col * s.dk + tile * 16 + hi * 4);
      o.qt[t] = *reinterpret_cast<const f32x4*>(unit + (CH + col) * s.dk + tile * 16 + hi * 4);
      o.kh[t] = *reinterpret_cast<const f32x4*>(kh + (tile * 16 + col) * CH + hi * 4);
      o.g[t] = *reinterpret_cast<const f32x4*>(g + tile * 16 + hi * 4);
    }
    o.t = *reinterpret_cast<const f32x4*>(tt + col * CH + hi * 4);
    o.qk = *reinterpret_cast<const f32x4*>(tt + CH * CH + col * CH + hi * 4);
#pragma unroll
    for (int r = 0; r < 4; ++r) o.v[r] = v[(hi * 4 + r) * s.dv + v0 + col];
  };
  auto step = [&](int c, const ChunkOperands<TPW>& now) {
    f32x4 pk = zero, pq = zero;
#pragma unroll
    for (int t = 0; t < TPW; ++t) {
      pk = mma16(now.kt[t], acc[t], pk);
      pq = mma16(now.qt[t], acc[t], pq);
    }
    const int buf = c & 1;
    part[buf][wave][0][lane] = pk;
    part[buf][wave][1][lane] = pq;
    lds_barrier();
    pk = (part[buf][0][0][lane] + part[buf][1][0][lane]) + (part[buf][2][0][lane] + part[buf][3][0][lane]);
    f32x4 rest;
#pragma unroll
    for (int r = 0; r < 4; ++r) rest[r] = now.v[r] - pk[r];
    const f32x4 u = mma16(now.t, rest, zero);
#pragma unroll
    for (int t = 0; t < TPW; ++t) {
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[t][r] *= now.g[t][r];
      // no branch around a product: the tile past the last one takes zeros
      const bool live = wave + t * 4 < n_tiles;
      f32x4 kh;
#pragma unroll
      for (int r = 0; r < 4; ++r) kh[r] = live ? now.kh[t][r] : 0.f;
      acc[t] = mma16(kh, u, acc[t]);
    }
    if (wave == 3) {  // the wave with the fewest tiles
      pq = (part[buf][0][1][lane] + part[buf][1][1][lane]) + (part[buf][2][1][lane] + part[buf][3][1][lane]);
      pq = mma16(now.qk, u, pq);
      const int row0 = tiles[2 * c], n = tiles[2 * c + 1];
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (hi * 4 + r < n && v0 + col < s.vdim)
          out[((size_t)(row0 + hi * 4 + r) * s.heads + h) * s.vdim + v0 + col] = pq[r];
    }
  };
  auto load_ahead = [&](int c, ChunkOperands<TPW>& o) { load(min(c, c1 - 1), o); };
  ChunkOperands<TPW> o0, o1, o2, o3;  // written out: an indexed array would not stay in registers
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
#pragma unroll
  for (int t = 0; t < TPW; ++t) {
    const int tile = wave + t * 4;
    if (tile < n_tiles)
#pragma unroll
      for (int r = 0; r < 4; ++r) st[(size_t)(tile * 16 + hi * 4 + r) * s.dv] = acc[t][r];
  }
}

// Grid: (sequences, channels / 256)
template <typename TY>
__global__ __launch_bounds__(256) void delta_conv_tail(
    const TY* __restrict__ y, int stride, const int* __restrict__ tiles, const int* __restrict__ bounds,
    const int* __restrict__ pos, const int* __restrict__ slot_of, float* __restrict__ conv, DeltaShape s) {
  const int seq = blockIdx.x, ch = blockIdx.y * 256 + threadIdx.x;
  if (ch >= s.channels() || bounds[seq] >= bounds[seq + 1]) return;
  const int slot = min(max(slot_of[seq], 0), s.slots - 1);
  const int first = tiles[2 * bounds[seq]], last = bounds[seq + 1] - 1;
  const int end = tiles[2 * last] + tiles[2 * last + 1];
  const int nk = s.kv_heads * s.dim;
  const int col = ch < nk ? s.oq + ch : ch < 2 * nk ? s.ok + ch - nk : s.ov + ch - 2 * nk;
  for (int row = max(first, end - s.taps); row < end; ++row)
    conv[((size_t)slot * s.taps + pos[row] % s.taps) * s.channels() + ch] = load_f32(y + (size_t)row * stride + col);
}

// out[t, h * vdim + c] = o / rms(o) * w * sigmoid(gate); 16 lanes per (token, head)
template <typename TO>
__global__ __launch_bounds__(256) void delta_norm_kernel(
    const float* __restrict__ o, const float* __restrict__ gate, const float* __restrict__ w, TO* __restrict__ out,
    int out_stride, int heads, int vdim, long total, float eps) {
  const long th = (long)blockIdx.x * 16 + threadIdx.x / 16;
  if (th >= total) return;  // all 16 lanes
  const int lane = threadIdx.x & 15;
  const float* src = o + th * vdim;
  const float* gs = gate + th * vdim;
  TO* dst = out + th / heads * out_stride + th % heads * vdim;
  float ss = 0.f;
  if (vdim % 8 == 0 && vdim <= 256) {
    float o8[2][8], g8[2][8];
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      const int c = lane * 8 + m * 128;
      if (c < vdim) {
        load8(src + c, o8[m]);
        load8(gs + c, g8[m]);
#pragma unroll
        for (int e = 0; e < 8; ++e) ss = fmaf(o8[m][e], o8[m][e], ss);
      }
    }
    const float inv = 1.f / sqrtf(group16_reduce_sum(ss) / vdim + eps);
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      const int c = lane * 8 + m * 128;
      if (c < vdim) {
#pragma unroll
        for (int e = 0; e < 8; ++e) o8[m][e] *= inv * w[c + e] / (1.f + expf(-g8[m][e]));
        store8(dst + c, o8[m]);
      }
    }
    return;
  }
  for (int c = lane; c < vdim; c += 16) ss = fmaf(src[c], src[c], ss);
  const float inv = 1.f / sqrtf(group16_reduce_sum(ss) / vdim + eps);
  for (int c = lane; c < vdim; c += 16) store_f32(dst + c, src[c] * inv * w[c] / (1.f + expf(-gs[c])));
}

// ----------------------------------------------------------------- decoding

struct LowRank {
  int a1, g1;          // first columns of the two inner projections
  int a_rank, g_rank;  // multiples of 8, zero-padded
};

// sum_r w[r] x[r] by 2 neighbouring lanes, the same value in both
template <typename TY, typename TW>
__device__ __forceinline__ float pair_dot(const TY* x, const TW* w, int rank, int part) {
  float s = 0.f;
#pragma unroll 8
  for (int r = part * 8; r < rank; r += 16) {
    float a[8], b[8];
    load8(w + r, a);
    load8(x + r, b);
#pragma unroll
    for (int e = 0; e < 8; ++e) s = fmaf(a[e], b[e], s);
  }
  return s + __shfl_xor(s, 1, WAVE);
}

// Grid: (tokens, heads); row t is sequence t's only one. 512 threads hold S, 4 columns
// and NR rows each.
template <typename TY, typename TW, int NR>
__global__ __launch_bounds__(512) void delta_decode_kernel(
    ConvInput<TY> in, float* __restrict__ conv_out, const TW* __restrict__ a2, const TW* __restrict__ g2, LowRank lr,
    const float* __restrict__ a_exp, const float* __restrict__ dt_bias, const float* __restrict__ norm_w,
    const int* __restrict__ pos, const int* __restrict__ slot_of,
    float* __restrict__ state, TY* __restrict__ out, int out_stride, DeltaShape s, float eps) {
  extern __shared__ float sm[];
  float* sq = sm;            // [dk]
  float* sk = sq + s.dk;     // [dk]
  float* sg = sk + s.dk;     // [dk] decay
  float* sv = sg + s.dk;     // [dv]
  float* gate = sv + s.dv;   // [dv]
  float* red = gate + s.dv;  // [2048]
  __shared__ float scal[3];
  const int tid = threadIdx.x, lane = tid & (WAVE - 1);
  const int row = blockIdx.x, h = blockIdx.y, group = s.heads / s.kv_heads, kvh = h / group;
  const int p = pos[row], slot = min(max(slot_of[row], 0), s.slots - 1);
  const TY* yr = in.y + (size_t)row * in.stride;

  // S is on its way while the vectors are made
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

  const int ring_row = p % s.taps;
#pragma unroll 1
  for (int i = tid; i < 2 * s.dk + s.dv; i += 512) {
    const int part = i < s.dk ? 0 : i < 2 * s.dk ? 1 : 2;
    const int c = i - part * s.dk;
    float x = 0.f;
    if (c < (part < 2 ? s.dim : s.vdim)) {
      const int at = part < 2 ? kvh * s.dim + c : h * s.vdim + c;
      const int col = (part == 0 ? s.oq : part == 1 ? s.ok : s.ov) + at;
      const int ch = part * s.kv_heads * s.dim + at;
      const float own = load_f32(yr + col);
      x = own * in.w[(s.taps - 1) * s.channels() + ch];
      const float* w = in.w + (s.taps - 1) * s.channels() + ch;
      const float* ring = in.state + (size_t)slot * s.taps * s.channels() + ch;
      for (int a0 = 1; a0 < s.taps; a0 += 4) {  // 4 loads on their way at once
        float v[4], wt[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int ago = a0 + e < s.taps ? a0 + e : 0;
          v[e] = ring[(ring_row >= ago ? ring_row - ago : ring_row - ago + s.taps) * s.channels()];
          wt[e] = w[-ago * s.channels()];
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) x = a0 + e < s.taps && a0 + e <= p ? fmaf(wt[e], v[e], x) : x;
      }
      x /= 1.f + expf(-x);
      // this row is read by no other workgroup, and not used above
      if (part == 2 || h == kvh * group)
        conv_out[((size_t)slot * s.taps + ring_row) * s.channels() + ch] = own;
    }
    (part == 0 ? sq : part == 1 ? sk : sv)[c] = x;
  }
#pragma unroll 1
  for (int i = tid; i < (s.dk + s.dv) * 2; i += 512) {
    const int part = i & 1;
    const bool decays = i < s.dk * 2;
    const int c = (i >> 1) - (decays ? 0 : s.dk), n = decays ? s.dim : s.vdim, at = h * n + min(c, n - 1);
    const int rank = decays ? lr.a_rank : lr.g_rank;
    const float z = pair_dot(yr + (decays ? lr.a1 : lr.g1), (decays ? a2 : g2) + (size_t)at * rank, rank, part);
    float g = 0.f;
    if (decays) g = exp2f(log_decay(z, dt_bias[at], a_exp[h]));
    else g = 1.f / (1.f + expf(-z));
    if (part == 0) (decays ? sg : gate)[c] = c < n ? g : 0.f;
  }
  __syncthreads();
  if (tid < 2 * WAVE) {
    const float* x = tid < WAVE ? sq : sk;
    float ss = 0.f;
    for (int c = lane; c < s.dim; c += WAVE) ss = fmaf(x[c], x[c], ss);
    ss = wave_reduce_sum(ss);
    if (lane == 0) scal[tid / WAVE] = 1.f / sqrtf(ss + 1e-6f);
  }
  if (tid == 2 * WAVE) scal[2] = 1.f / (1.f + expf(-load_f32(yr + s.ob + h)));
  __syncthreads();
  const float qn = scal[0] / sqrtf((float)s.dim), kn = scal[1], beta = scal[2];

  f32x4 sum = {0.f, 0.f, 0.f, 0.f};
  if (rg < rpp) {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int c = rg + i * rpp;
      if (c >= s.dk) break;
      const float g = sg[c], k = sk[c] * kn;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        acc[i][e] *= g;
        sum[e] = fmaf(acc[i][e], k, sum[e]);
      }
    }
    *reinterpret_cast<f32x4*>(&red[rg * s.dv + vc]) = sum;
  }
  __syncthreads();
  for (int c = tid; c < s.dv; c += 512) {
    float t = 0.f;
    for (int r = 0; r < rpp; ++r) t += red[r * s.dv + c];
    sv[c] = beta * (sv[c] - t);  // u
  }
  __syncthreads();
  if (rg < rpp) {
    const f32x4 u = *reinterpret_cast<const f32x4*>(&sv[vc]);
    sum = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int c = rg + i * rpp;
      if (c >= s.dk) break;
      const float k = sk[c] * kn, q = sq[c] * qn;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        acc[i][e] = fmaf(k, u[e], acc[i][e]);
        sum[e] = fmaf(acc[i][e], q, sum[e]);
      }
      *reinterpret_cast<f32x4*>(st + (size_t)c * s.dv) = acc[i];
    }
    *reinterpret_cast<f32x4*>(&red[rg * s.dv + vc]) = sum;
  }
  __syncthreads();
  float mine = 0.f;
  for (int c = tid; c < s.dv; c += 512) {
    float t = 0.f;
    for (int r = 0; r < rpp; ++r) t += red[r * s.dv + c];
    sv[c] = t;
    mine = fmaf(t, t, mine);
  }
  mine = wave_reduce_sum(mine);
  __shared__ float wsum[8];
  if (lane == 0) wsum[tid / WAVE] = mine;
  __syncthreads();
  float ss = 0.f;
#pragma unroll
  for (int w = 0; w < 8; ++w) ss += wsum[w];
  const float inv = 1.f / sqrtf(ss / s.vdim + eps);
  for (int c = tid; c < s.vdim; c += 512)
    store_f32(out + (size_t)row * out_stride + h * s.vdim + c, sv[c] * inv * norm_w[c] * gate[c]);
}

// ------------------------------------------------------------------- host

// cols: first columns of q, k, v, beta in the projection
static DeltaShape delta_shape(const torch::Tensor& y, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim,
                              const std::vector<int64_t>& cols, const torch::Tensor& conv_w, const torch::Tensor& delta,
                              const torch::Tensor& conv) {
  TORCH_CHECK(kv_heads >= 1 && heads % kv_heads == 0 && dim >= 1 && vdim >= 1 && cols.size() == 4);
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous());
  TORCH_CHECK(y.dtype() == torch::kFloat32 || y.dtype() == torch::kBFloat16);
  DeltaShape s;
  s.heads = heads, s.kv_heads = kv_heads, s.dim = dim, s.vdim = vdim;
  s.dk = (dim + 15) / 16 * 16, s.dv = (vdim + 15) / 16 * 16;
  s.oq = cols[0], s.ok = cols[1], s.ov = cols[2], s.ob = cols[3];
  const long width = y.size(1);
  TORCH_CHECK(cols[0] >= 0 && cols[0] + kv_heads * dim <= width && cols[1] >= 0 && cols[1] + kv_heads * dim <= width &&
              cols[2] >= 0 && cols[2] + heads * vdim <= width && cols[3] >= 0 && cols[3] + heads <= width);
  TORCH_CHECK(conv_w.dim() == 2 && conv_w.size(1) == s.channels());
  s.taps = conv_w.size(0);
  check_f32(conv_w, (long)s.channels() * s.taps, "convolution weights");
  TORCH_CHECK(delta.dim() == 4 && conv.dim() == 3);
  s.slots = delta.size(0);
  check_f32(delta, (long)s.slots * heads * s.dk * s.dv, "delta state");
  TORCH_CHECK(conv.size(0) == s.slots && conv.size(1) == s.taps && conv.size(2) == s.channels(), "conv state");
  check_f32(conv, conv.numel(), "conv state");
  return s;
}

// Rows of any number of sequences in chunks of 16; returns o [T, H * vdim] 32-bit,
// not yet normed. Updates both states.
torch::Tensor delta_prefill(
    torch::Tensor y, torch::Tensor a, torch::Tensor conv_w, torch::Tensor a_exp, torch::Tensor dt_bias,
    torch::Tensor tiles,   // [n, 2] runs of at most 16 rows
    torch::Tensor bounds,  // [S + 1] runs of each sequence
    torch::Tensor pos, torch::Tensor owner, torch::Tensor slot, torch::Tensor delta, torch::Tensor conv, int64_t heads,
    int64_t kv_heads, int64_t dim, int64_t vdim, std::vector<int64_t> cols) {
  const DeltaShape s = delta_shape(y, heads, kv_heads, dim, vdim, cols, conv_w, delta, conv);
  const long t = y.size(0), chunks = tiles.size(0), seqs = bounds.numel() - 1;
  check_f32(a, t * heads * dim, "decay projection");
  check_f32(a_exp, heads, "decay rates");
  check_f32(dt_bias, heads * dim, "decay bias");
  check_i32(tiles, 2 * chunks, "chunks");
  check_i32(bounds, seqs + 1, "chunk bounds");
  check_i32(pos, t, "positions");
  check_i32(owner, t, "owners");
  check_i32(slot, seqs, "slots");
  TORCH_CHECK(s.dk <= 512 && s.heads <= 65535 && seqs <= 65535, "key size ", dim, " is not supported");
  auto out = torch::empty({t, heads * vdim}, a.options());
  if (t == 0) return out;
  auto ws = torch::empty({(long)(chunks * heads * unit_size(s.dk, s.dv))}, a.options());
  auto stream = at::cuda::getCurrentCUDAStream();
  const size_t lds = ((size_t)3 * CH * (s.dk + 4) + CH * 17 + CH) * 4;
  const bool yf = y.dtype() == torch::kFloat32;
  const int* tp = tiles.data_ptr<int>();
  const int *bp = bounds.data_ptr<int>(), *pp = pos.data_ptr<int>(), *op = owner.data_ptr<int>(), *sp = slot.data_ptr<int>();
  const int stride = y.size(1);
  const dim3 tail_grid(seqs, (s.channels() + 255) / 256);
#define DC(TY, BY8, YP)                                                                                               \
  do {                                                                                                                \
    if (lds > 65536) {                                                                                                \
      const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&delta_chunk_kernel<TY, BY8>),           \
                                               hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);                 \
      TORCH_CHECK(e == hipSuccess, "LDS request refused: ", hipGetErrorString(e));                                    \
    }                                                                                                                 \
    const ConvInput<TY> in{YP, stride, conv_w.data_ptr<float>(), conv.data_ptr<float>()};                             \
    delta_chunk_kernel<TY, BY8><<<dim3(chunks, heads), 256, lds, stream>>>(in, a.data_ptr<float>(), a_exp.data_ptr<float>(), \
        dt_bias.data_ptr<float>(), tp, bp, pp, op, sp, s, ws.data_ptr<float>());                                      \
    HIP_CHECK_LAST();                                                                                                 \
    delta_conv_tail<TY><<<tail_grid, 256, 0, stream>>>(YP, stride, tp, bp, pp, sp, conv.data_ptr<float>(), s);        \
  } while (0)
  bool by8 = dim % 8 == 0 && vdim % 8 == 0 && stride % 8 == 0;
  for (int i = 0; i < 3; ++i) by8 = by8 && cols[i] % 8 == 0;
  for (const auto& p : {y, a, conv_w, dt_bias, conv}) by8 = by8 && reinterpret_cast<uintptr_t>(p.data_ptr()) % 16 == 0;
  if (yf && by8) DC(float, true, y.data_ptr<float>());
  else if (yf) DC(float, false, y.data_ptr<float>());
  else if (by8) DC(unsigned short, true, BF16P(y));
  else DC(unsigned short, false, BF16P(y));
#undef DC
  HIP_CHECK_LAST();
  const dim3 grid(heads, s.dv / 16, seqs);
  const int tpw = (s.dk / 16 + 3) / 4;
#define DS(N)                                                                                                         \
  delta_scan_kernel<N><<<grid, 256, 0, stream>>>(ws.data_ptr<float>(), tp, bp, pp, sp, delta.data_ptr<float>(),       \
                                                 out.data_ptr<float>(), s)
  if (tpw <= 1) DS(1);
  else if (tpw <= 2) DS(2);
  else if (tpw <= 4) DS(4);
  else DS(8);
#undef DS
  HIP_CHECK_LAST();
  return out;
}

// o, gate [T, H * vdim] 32-bit -> [T, width], zero past H * vdim
torch::Tensor delta_norm(torch::Tensor o, torch::Tensor gate, torch::Tensor w, int64_t heads, int64_t width, bool f32,
                         double eps) {
  const long t = o.size(0), vdim = w.numel();
  check_f32(o, t * heads * vdim, "delta output");
  check_f32(gate, t * heads * vdim, "delta gate");
  check_f32(w, vdim, "delta norm");
  TORCH_CHECK(width >= heads * vdim && (vdim % 8 || width % 8 == 0));
  const auto opt = o.options().dtype(f32 ? torch::kFloat32 : torch::kBFloat16);
  auto out = width == heads * vdim ? torch::empty({t, width}, opt) : torch::zeros({t, width}, opt);
  if (t == 0) return out;
  const long total = t * heads;
  auto stream = at::cuda::getCurrentCUDAStream();
#define DN(TO, OP)                                                                                              \
  delta_norm_kernel<TO><<<(total + 15) / 16, 256, 0, stream>>>(o.data_ptr<float>(), gate.data_ptr<float>(),       \
      w.data_ptr<float>(), OP, (int)width, (int)heads, (int)vdim, total, (float)eps)
  if (f32) DN(float, out.data_ptr<float>());
  else DN(unsigned short, BF16P(out));
#undef DN
  HIP_CHECK_LAST();
  return out;
}

// rows of S per thread in the decoding kernel, 0 if it does not take these sizes
static int decode_rows(const DeltaShape& s) {
  if (s.dv > 2048) return 0;
  const int rpp = 512 / (s.dv / 4), need = (s.dk + rpp - 1) / rpp;
  return need <= 4 ? 4 : need <= 8 ? 8 : need <= 16 ? 16 : need <= 32 ? 32 : 0;
}

bool delta_decodes(int64_t dim, int64_t vdim) {
  DeltaShape s;
  s.dk = (dim + 15) / 16 * 16, s.dv = (vdim + 15) / 16 * 16;
  return decode_rows(s) > 0 && (3 * s.dk + 2 * s.dv + 2048) * 4 <= 60000;
}

// One row per sequence; returns [T, width] in y's dtype, normed and gated.
torch::Tensor delta_decode(
    torch::Tensor y, torch::Tensor conv_w, torch::Tensor a2, torch::Tensor g2, int64_t a1_col, int64_t g1_col,
    torch::Tensor a_exp, torch::Tensor dt_bias, torch::Tensor norm_w, torch::Tensor pos, torch::Tensor slot,
    torch::Tensor delta, torch::Tensor conv, int64_t heads, int64_t kv_heads, int64_t dim,
    int64_t vdim, std::vector<int64_t> cols, int64_t width, double eps) {
  const DeltaShape s = delta_shape(y, heads, kv_heads, dim, vdim, cols, conv_w, delta, conv);
  const long t = y.size(0);
  const int stride = y.size(1);
  check_f32(a_exp, heads, "decay rates");
  check_f32(dt_bias, heads * dim, "decay bias");
  check_f32(norm_w, vdim, "delta norm");
  check_i32(pos, t, "positions");
  TORCH_CHECK(slot.numel() == t, "one row per sequence");
  check_i32(slot, t, "slots");
  const bool yf = y.dtype() == torch::kFloat32, wf = a2.dtype() == torch::kFloat32;
  for (const auto& w : {a2, g2})
    TORCH_CHECK(w.is_cuda() && w.dim() == 2 && w.is_contiguous() && w.size(1) % 8 == 0 &&
                w.dtype() == (wf ? torch::kFloat32 : torch::kBFloat16), "low-rank projections");
  TORCH_CHECK(a2.size(0) == heads * dim && g2.size(0) == heads * vdim && (yf || !wf));
  const LowRank lr{(int)a1_col, (int)g1_col, (int)a2.size(1), (int)g2.size(1)};
  TORCH_CHECK(a1_col % 8 == 0 && g1_col % 8 == 0 && stride % 8 == 0, "low-rank columns are read in groups of 8");
  TORCH_CHECK(a1_col >= 0 && a1_col + lr.a_rank <= y.size(1) && g1_col >= 0 && g1_col + lr.g_rank <= y.size(1));
  const int nr = decode_rows(s);
  TORCH_CHECK(delta_decodes(dim, vdim), "head sizes ", dim, " and ", vdim, " are not supported");
  TORCH_CHECK(width >= heads * vdim && heads <= 65535);
  auto out = width == heads * vdim ? torch::empty({t, width}, y.options()) : torch::zeros({t, width}, y.options());
  if (t == 0) return out;
  auto stream = at::cuda::getCurrentCUDAStream();
  const size_t lds = (size_t)(3 * s.dk + 2 * s.dv + 2048) * 4;
#define DD(TY, TW, N, YP, OP, A2, G2)                                                                              \
  delta_decode_kernel<TY, TW, N><<<dim3(t, heads), 512, lds, stream>>>(                                            \
      ConvInput<TY>{YP, stride, conv_w.data_ptr<float>(), conv.data_ptr<float>()}, conv.data_ptr<float>(), A2, G2, \
      lr, a_exp.data_ptr<float>(), dt_bias.data_ptr<float>(), norm_w.data_ptr<float>(), pos.data_ptr<int>(),       \
      slot.data_ptr<int>(), delta.data_ptr<float>(), OP, (int)width, s, (float)eps)
#define DDN(TY, TW, YP, OP, A2, G2)                      \
  do {                                                   \
    if (nr == 4) DD(TY, TW, 4, YP, OP, A2, G2);          \
    else if (nr == 8) DD(TY, TW, 8, YP, OP, A2, G2);     \
    else if (nr == 16) DD(TY, TW, 16, YP, OP, A2, G2);   \
    else DD(TY, TW, 32, YP, OP, A2, G2);                 \
  } while (0)
  if (yf && wf) DDN(float, float, y.data_ptr<float>(), out.data_ptr<float>(), a2.data_ptr<float>(), g2.data_ptr<float>());
  else if (yf) DDN(float, unsigned short, y.data_ptr<float>(), out.data_ptr<float>(), BF16P(a2), BF16P(g2));
  else DDN(unsigned short, unsigned short, BF16P(y), BF16P(out), BF16P(a2), BF16P(g2));
#undef DDN
#undef DD
  HIP_CHECK_LAST();
  return out;
}
