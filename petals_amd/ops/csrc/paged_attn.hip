// Attention over paged keys and values for CDNA4 (gfx950): grouped heads with
// separate key and value sizes, sliding window, a bias per head that grows with
// the distance, one learned entry of the softmax's denominator per head (a sink),
// and a sigmoid gate on the output.
//
// A token's cache row is [G heads of DK keys | G heads of DV values], DK a
// multiple of 32 and DV of 16 (padded with zeros when weights are packed).
//
//   paged_attn_kernel   MFMA flash kernel for prompts and portions: 4 waves of 16
//                       (token, head) rows share double-buffered key/value tiles
//   paged_attn_decode   few rows per kv head: every wave takes tiles of its own,
//                       keys straight from memory, merged through LDS at the end
//   paged_attn_combine  merges key splits
//   paged_attn_simple   any size, 32-bit or bf16 storage
//   attn_prepare        bias, query temperature, value mixing; writes the cache
//
// Every page index is checked against the pool before it is used.

#include "common.h"
#include "paged.h"
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>

#define KVT 32   // keys per tile; tiles are aligned, so one lies in one page
#define TPAD 16  // LDS row padding (elements)
#define LOG2E 1.4426950408889634f

struct AttnShape {
  int heads, kv_heads, dk, dv;  // padded head sizes
  int window;                   // 0: everything before
  float scale;
  const float* slopes;  // [heads] or null
  const float* sink;    // [heads] or null
};

// where the result goes: out[t, head * dv + c] = o * sigmoid(gate[t, head * dv + c])
struct GatedOut {
  void* out;         // [T, heads * dv]
  const void* gate;  // row stride gate_stride, or null
  long gate_stride;
  bool f32;          // both in 32-bit, else bf16
};

__device__ __forceinline__ void write_gated(const GatedOut& g, const AttnShape& a, size_t tok, int head, int c, float v) {
  const int col = head * a.dv + c;
  if (g.gate) {
    const size_t at = tok * g.gate_stride + col;
    const float z = g.f32 ? reinterpret_cast<const float*>(g.gate)[at]
                          : bf16_to_f32(reinterpret_cast<const unsigned short*>(g.gate)[at]);
    v /= 1.f + expf(-z);
  }
  const size_t to = tok * (size_t)(a.heads * a.dv) + col;
  if (g.f32) reinterpret_cast<float*>(g.out)[to] = v;
  else reinterpret_cast<unsigned short*>(g.out)[to] = f32_to_bf16(v);
}

__device__ __forceinline__ void wave_lds_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// Scores of a 16-row x 32-key tile (C layout: key col of block nb, rows hi*4+r)
// -> probabilities; updates the running maximum and this lane's share of the sum.
struct SoftmaxRows {
  float m[4], l[4], slope[4];  // slope in log2 units
  int pos[4], lo[4];           // the row sees keys in [lo, pos]
};

__device__ __forceinline__ void softmax_tile(
    SoftmaxRows& w, const f32x4* s_acc, int j0, int col, int j_end, bool interior, float scale_l2, float corr[4],
    float p[2][4]) {
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    float s[2];
#pragma unroll
    for (int nb = 0; nb < 2; ++nb)
      s[nb] = s_acc[nb][r] * scale_l2 - w.slope[r] * (float)(w.pos[r] - (j0 + nb * 16 + col));
    // masking and the running max stay in separate loops (see prefill_attn.hip)
    if (!interior) {
#pragma unroll
      for (int nb = 0; nb < 2; ++nb) {
        const int key = j0 + nb * 16 + col;
        if (key >= j_end || key > w.pos[r] || key < w.lo[r]) s[nb] = NEG_SENTINEL;
      }
    }
    float mx = fmaxf(s[0], s[1]);
#pragma unroll
    for (int off = 8; off > 0; off >>= 1) mx = fmaxf(mx, __shfl_xor(mx, off, WAVE));
    const float m_new = fmaxf(w.m[r], mx);
    corr[r] = (w.m[r] <= NEG_THRESHOLD) ? 0.f : exp2f(w.m[r] - m_new);
#pragma unroll
    for (int nb = 0; nb < 2; ++nb) p[nb][r] = (s[nb] <= NEG_THRESHOLD) ? 0.f : exp2f(s[nb] - m_new);
    w.l[r] = w.l[r] * corr[r] + (p[0][r] + p[1][r]);
    w.m[r] = m_new;
  }
}

// ------------------------------------------------------------ MFMA kernel

// RC: 32-wide chunks of the key size, VB: 16-wide blocks of the value size, at
// least as many as there are: tiles are filled up with zeros, so that no branch
// stands between products.
// Grid: (token runs, kv heads x groups of 64 rows, key splits).
template <int RC, int VB>
__global__ __launch_bounds__(256) void paged_attn_kernel(
    const unsigned short* __restrict__ q,      // [T, H, dk]
    const unsigned short* __restrict__ cache,  // [pages, PAGE, G * (dk + dv)]
    GatedOut g,                                // n_splits == 1
    float* __restrict__ part_o,                // [n_splits, T*H, dv]
    float* __restrict__ part_ml,               // [n_splits, T*H, 2]
    const int* __restrict__ tiles,             // [n, 2] first token, token count
    PagedRows b, AttnShape a, int total_tokens, int n_splits) {
  constexpr int KROW = RC * 32 + TPAD, VROW = VB * 16 + TPAD;
  constexpr int K8 = RC * 4, V8 = VB * 2;                    // 16-byte groups of a row
  constexpr int K_LOADS = KVT * K8, LOADS = KVT * (K8 + V8);
  constexpr int NLD = (LOADS + 255) / 256;                   // per thread
  const int tok0 = tiles[2 * blockIdx.x];
  const int ntok = tiles[2 * blockIdx.x + 1];
  const int group = a.heads / a.kv_heads;
  const int rows = ntok * group;
  const int kvh = blockIdx.y % a.kv_heads;
  const int g0 = blockIdx.y / a.kv_heads * 64;
  if (g0 >= rows) return;  // uniform over the workgroup
  const int g1 = min(g0 + 64, rows);

  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & (WAVE - 1);
  const int col = lane & 15, hi = lane >> 4;
  const int r0 = g0 + wave * 16;

  extern __shared__ unsigned short smem[];
  unsigned short* p_lds = smem + 2 * KVT * (KROW + VROW) + wave * 16 * (KVT + 8);

  const int seq = b.owner[tok0];
  const int first_pos = b.pos[tok0 + g0 / group];
  const int last_pos = b.pos[tok0 + (g1 - 1) / group];
  const int key_lo = a.window > 0 ? max(0, first_pos - a.window + 1) / KVT * KVT : 0;
  const int key_hi = last_pos + 1;
  const int n_tiles = (key_hi - key_lo + KVT - 1) / KVT;
  const int per_split = (n_tiles + n_splits - 1) / n_splits;
  const int j_begin = key_lo + blockIdx.z * per_split * KVT;
  const int j_end = min(key_hi, j_begin + per_split * KVT);

  bf16x8 q_frag[RC];
  {
    const int row = r0 + col;
    const size_t at = ((size_t)(tok0 + row / group) * a.heads + kvh * group + row % group) * a.dk;
#pragma unroll
    for (int kc = 0; kc < RC; ++kc)
      q_frag[kc] = row < rows && kc * 32 < a.dk ? *reinterpret_cast<const bf16x8*>(q + at + kc * 32 + hi * 8)
                                                : bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
  }

  f32x4 acc_o[VB];
  SoftmaxRows w;
#pragma unroll
  for (int d = 0; d < VB; ++d) acc_o[d] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int row = r0 + hi * 4 + r;
    w.m[r] = NEG_SENTINEL;
    w.l[r] = 0.f;
    w.pos[r] = row < rows ? b.pos[tok0 + row / group] : -1;  // -1: sees nothing
    w.lo[r] = a.window > 0 ? w.pos[r] - a.window + 1 : 0;
    w.slope[r] = row < rows && a.slopes ? a.slopes[kvh * group + row % group] * LOG2E : 0.f;
  }
  // keys that every row of this wave sees: [all_lo, all_hi]; those that some row sees: [any_lo, any_hi]
  const bool full_wave = r0 + 16 <= rows;
  const int wave_first = r0 < rows ? b.pos[tok0 + r0 / group] : -1;
  const int wave_last = r0 < rows ? b.pos[tok0 + (min(r0 + 16, rows) - 1) / group] : -1;
  const int all_hi = full_wave ? wave_first : -1;
  const int all_lo = full_wave && a.window > 0 ? wave_last - a.window + 1 : 0;
  const int any_hi = wave_last, any_lo = a.window > 0 ? wave_first - a.window + 1 : 0;

  const int width = a.kv_heads * (a.dk + a.dv);
  bf16x8 next[NLD];
  // rows of tile j0 that lie in [0, j_end); zero elsewhere
  auto fetch = [&](int j0) {
    const long at = cache_row(b, seq, j0);
#pragma unroll
    for (int i = 0; i < NLD; ++i) {
      const int idx = tid + i * 256;
      next[i] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
      if (LOADS % 256 == 0 || idx < LOADS) {
        const bool is_v = idx >= K_LOADS;
        const int row = is_v ? (idx - K_LOADS) / V8 : idx / K8;
        const int c8 = (is_v ? (idx - K_LOADS) % V8 : idx % K8) * 8;
        const int c = is_v ? a.kv_heads * a.dk + kvh * a.dv + c8 : kvh * a.dk + c8;
        if (at >= 0 && j0 + row < j_end && c8 < (is_v ? a.dv : a.dk))
          next[i] = *reinterpret_cast<const bf16x8*>(cache + ((size_t)at + row) * width + c);
      }
    }
  };
  auto stage = [&](unsigned short* buf) {
#pragma unroll
    for (int i = 0; i < NLD; ++i) {
      const int idx = tid + i * 256;
      if (LOADS % 256 == 0 || idx < LOADS) {
        const bool is_v = idx >= K_LOADS;
        const int row = is_v ? (idx - K_LOADS) / V8 : idx / K8;
        const int c8 = (is_v ? (idx - K_LOADS) % V8 : idx % K8) * 8;
        unsigned short* dst = is_v ? buf + KVT * KROW + row * VROW + c8 : buf + row * KROW + c8;
        *reinterpret_cast<bf16x8*>(dst) = next[i];
      }
    }
  };

  const float scale_l2 = a.scale * LOG2E;
  if (j_begin < j_end) {
    fetch(j_begin);
    stage(smem);
  }
  __syncthreads();
  int which = 0;
  for (int j0 = j_begin; j0 < j_end; j0 += KVT, which ^= 1) {
    const unsigned short* k_lds = smem + which * KVT * (KROW + VROW);
    const bool more = j0 + KVT < j_end;
    if (more) fetch(j0 + KVT);
    if (j0 <= any_hi && j0 + KVT > any_lo) {  // uniform over the wave
      f32x4 s_acc[2];
#pragma unroll
      for (int nb = 0; nb < 2; ++nb) {
        s_acc[nb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kc = 0; kc < RC; ++kc) {
          const bf16x8 kt = *reinterpret_cast<const bf16x8*>(&k_lds[(nb * 16 + col) * KROW + kc * 32 + hi * 8]);
          s_acc[nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(q_frag[kc], kt, s_acc[nb], 0, 0, 0);
        }
      }
      const bool interior = j0 >= all_lo && j0 + KVT - 1 <= all_hi && j0 + KVT <= j_end;
      float corr[4], p[2][4];
      softmax_tile(w, s_acc, j0, col, j_end, interior, scale_l2, corr, p);
      // P to A-fragment layout through this wave's own LDS
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int nb = 0; nb < 2; ++nb) p_lds[(hi * 4 + r) * (KVT + 8) + nb * 16 + col] = f32_to_bf16(p[nb][r]);
      wave_lds_fence();
      const bf16x8 p_frag = *reinterpret_cast<const bf16x8*>(&p_lds[col * (KVT + 8) + hi * 8]);
      const unsigned short* v_lds = k_lds + KVT * KROW + (hi * 8 + col / 4) * VROW + (col & 3) * 4;
#pragma unroll
      for (int d = 0; d < VB; ++d) {
#pragma unroll
        for (int r = 0; r < 4; ++r) acc_o[d][r] *= corr[r];
        acc_o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(p_frag, load_keys(v_lds + d * 16, VROW), acc_o[d], 0, 0, 0);
      }
    }
    if (more) stage(smem + (which ^ 1) * KVT * (KROW + VROW));
    __syncthreads();
  }

#pragma unroll
  for (int r = 0; r < 4; ++r) {
    float l = w.l[r];
#pragma unroll
    for (int off = 8; off > 0; off >>= 1) l += __shfl_xor(l, off, WAVE);
    const int row = r0 + hi * 4 + r;
    if (row >= rows) continue;
    const size_t tok = tok0 + row / group;
    const int head = kvh * group + row % group;
    if (n_splits == 1) {
      float scale = 1.f;
      if (a.sink) {
        const float z = a.sink[head] * LOG2E, m = fmaxf(w.m[r], z);
        scale = exp2f(w.m[r] - m);
        l = l * scale + exp2f(z - m);
      }
      const float inv_l = l > 0.f ? scale / l : 0.f;
#pragma unroll
      for (int d = 0; d < VB; ++d)
        if (d * 16 < a.dv) write_gated(g, a, tok, head, d * 16 + col, acc_o[d][r] * inv_l);
    } else {
      const size_t at = ((size_t)blockIdx.z * total_tokens + tok) * a.heads + head;
#pragma unroll
      for (int d = 0; d < VB; ++d)
        if (d * 16 < a.dv) part_o[at * a.dv + d * 16 + col] = acc_o[d][r];
      if (col == 0) {
        part_ml[at * 2] = w.m[r];
        part_ml[at * 2 + 1] = l;
      }
    }
  }
}

// --------------------------------------------------------------- few rows

// One token and one kv head with at most 16 query heads. Grid: (tokens, kv
// heads, key splits); the 4 waves of a workgroup take every fourth tile.
template <int RC, int VB>
__global__ __launch_bounds__(256) void paged_attn_decode(
    const unsigned short* __restrict__ q, const unsigned short* __restrict__ cache, GatedOut g,
    float* __restrict__ part_o, float* __restrict__ part_ml, PagedRows b, AttnShape a, int total_tokens, int n_splits) {
  constexpr int VROW = VB * 16 + TPAD;
  constexpr int V8 = VB * 2;                // 16-byte groups of a row
  constexpr int NLD = V8 * KVT / WAVE;      // value loads per lane
  const int tok = blockIdx.x, kvh = blockIdx.y;
  const int group = a.heads / a.kv_heads;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & (WAVE - 1);
  const int col = lane & 15, hi = lane >> 4;
  extern __shared__ unsigned short smem[];
  unsigned short* v_tile = smem + wave * (KVT * VROW + 16 * (KVT + 8));
  unsigned short* p_lds = v_tile + KVT * VROW;

  const int seq = b.owner[tok], pos = b.pos[tok];
  const int key_lo = a.window > 0 ? max(0, pos - a.window + 1) / KVT * KVT : 0;
  const int n_tiles = (pos + 1 - key_lo + KVT - 1) / KVT;
  const int per_split = (n_tiles + n_splits - 1) / n_splits;
  const int j_begin = key_lo + blockIdx.z * per_split * KVT;
  const int j_end = min(pos + 1, j_begin + per_split * KVT);

  bf16x8 q_frag[RC];
  const size_t q_at = ((size_t)tok * a.heads + kvh * group + col) * a.dk;
#pragma unroll
  for (int kc = 0; kc < RC; ++kc)
    q_frag[kc] = col < group && kc * 32 < a.dk ? *reinterpret_cast<const bf16x8*>(q + q_at + kc * 32 + hi * 8)
                                               : bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
  f32x4 acc_o[VB];
  SoftmaxRows w;
#pragma unroll
  for (int d = 0; d < VB; ++d) acc_o[d] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int row = hi * 4 + r;
    w.m[r] = NEG_SENTINEL;
    w.l[r] = 0.f;
    w.pos[r] = row < group ? pos : -1;
    w.lo[r] = a.window > 0 ? pos - a.window + 1 : 0;
    w.slope[r] = row < group && a.slopes ? a.slopes[kvh * group + row] * LOG2E : 0.f;
  }
  const int width = a.kv_heads * (a.dk + a.dv);
  const float scale_l2 = a.scale * LOG2E;
  for (int j0 = j_begin + wave * KVT; j0 < j_end; j0 += 4 * KVT) {
    const long at = cache_row(b, seq, j0);
    bf16x8 vals[NLD], kt[2][RC];
#pragma unroll
    for (int nb = 0; nb < 2; ++nb)
#pragma unroll
      for (int kc = 0; kc < RC; ++kc) {
        const int row = nb * 16 + col;
        kt[nb][kc] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
        if (kc * 32 < a.dk && at >= 0 && j0 + row < j_end)
          kt[nb][kc] = *reinterpret_cast<const bf16x8*>(
              cache + ((size_t)at + row) * width + kvh * a.dk + kc * 32 + hi * 8);
      }
#pragma unroll
    for (int i = 0; i < NLD; ++i) {
      const int idx = lane + i * WAVE, row = idx / V8, c8 = idx % V8 * 8;
      vals[i] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
      if (at >= 0 && j0 + row < j_end && c8 < a.dv)
        vals[i] = *reinterpret_cast<const bf16x8*>(
            cache + ((size_t)at + row) * width + a.kv_heads * a.dk + kvh * a.dv + c8);
    }
    f32x4 s_acc[2];
#pragma unroll
    for (int nb = 0; nb < 2; ++nb) {
      s_acc[nb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kc = 0; kc < RC; ++kc)
        s_acc[nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(q_frag[kc], kt[nb][kc], s_acc[nb], 0, 0, 0);
    }
    float corr[4], p[2][4];
    softmax_tile(w, s_acc, j0, col, j_end, false, scale_l2, corr, p);
    wave_lds_fence();  // the last tile's reads are done
#pragma unroll
    for (int i = 0; i < NLD; ++i) {
      const int idx = lane + i * WAVE, row = idx / V8, c8 = idx % V8 * 8;
      *reinterpret_cast<bf16x8*>(&v_tile[row * VROW + c8]) = vals[i];
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int nb = 0; nb < 2; ++nb) p_lds[(hi * 4 + r) * (KVT + 8) + nb * 16 + col] = f32_to_bf16(p[nb][r]);
    wave_lds_fence();
    const bf16x8 p_frag = *reinterpret_cast<const bf16x8*>(&p_lds[col * (KVT + 8) + hi * 8]);
    const unsigned short* v_lds = v_tile + (hi * 8 + col / 4) * VROW + (col & 3) * 4;
#pragma unroll
    for (int d = 0; d < VB; ++d) {
#pragma unroll
      for (int r = 0; r < 4; ++r) acc_o[d][r] *= corr[r];
      acc_o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(p_frag, load_keys(v_lds + d * 16, VROW), acc_o[d], 0, 0, 0);
    }
  }
  // merge the waves: [4][group] maxima and sums, then [4][group][dv] weighted sums
  __syncthreads();
  float* ml = reinterpret_cast<float*>(smem);   // [4][16][2]
  float* os = ml + 4 * 16 * 2;                  // [4][group][dv]
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    float l = w.l[r];
#pragma unroll
    for (int off = 8; off > 0; off >>= 1) l += __shfl_xor(l, off, WAVE);
    const int row = hi * 4 + r;
    if (row >= group) continue;
    if (col == 0) {
      ml[(wave * 16 + row) * 2] = w.m[r];
      ml[(wave * 16 + row) * 2 + 1] = l;
    }
#pragma unroll
    for (int d = 0; d < VB; ++d)
      if (d * 16 < a.dv) os[(wave * group + row) * a.dv + d * 16 + col] = acc_o[d][r];
  }
  __syncthreads();
  for (int i = tid; i < group * a.dv; i += 256) {
    const int row = i / a.dv, c = i - row * a.dv, head = kvh * group + row;
    float m = NEG_SENTINEL;
#pragma unroll
    for (int u = 0; u < 4; ++u) m = fmaxf(m, ml[(u * 16 + row) * 2]);
    const float seen = m;
    if (n_splits == 1 && a.sink) m = fmaxf(m, a.sink[head] * LOG2E);
    float l = 0.f, o = 0.f;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const float mu = ml[(u * 16 + row) * 2];
      const float e = mu > NEG_THRESHOLD ? exp2f(mu - m) : 0.f;
      l = fmaf(e, ml[(u * 16 + row) * 2 + 1], l);
      o = fmaf(e, os[(u * group + row) * a.dv + c], o);
    }
    if (n_splits == 1) {
      if (a.sink) l += exp2f(a.sink[head] * LOG2E - m);
      write_gated(g, a, tok, head, c, l > 0.f ? o / l : 0.f);
    } else {
      const size_t at = ((size_t)blockIdx.z * total_tokens + tok) * a.heads + head;
      part_o[at * a.dv + c] = o;
      if (c == 0) {
        part_ml[at * 2] = seen;
        part_ml[at * 2 + 1] = l;
      }
    }
  }
}

// one workgroup per (token, head) row
__global__ __launch_bounds__(128) void paged_attn_combine(
    const float* __restrict__ part_o, const float* __restrict__ part_ml, GatedOut g, AttnShape a, int n_rows,
    int n_splits) {
  __shared__ float share[WAVE];  // weight of each split in the row
  const int row = blockIdx.x, head = row % a.heads;
  if (threadIdx.x < WAVE) {
    const int s = threadIdx.x;
    float m = NEG_SENTINEL, l = 0.f;
    if (s < n_splits) {
      m = part_ml[((size_t)s * n_rows + row) * 2];
      l = part_ml[((size_t)s * n_rows + row) * 2 + 1];
    }
    float mx = wave_reduce_max(m);
    if (a.sink) mx = fmaxf(mx, a.sink[head] * LOG2E);
    const float w = m > NEG_THRESHOLD ? exp2f(m - mx) : 0.f;
    float sum = wave_reduce_sum(w * l);
    if (a.sink) sum += exp2f(a.sink[head] * LOG2E - mx);
    share[s] = sum > 0.f ? w / sum : 0.f;
  }
  __syncthreads();
  for (int d = threadIdx.x; d < a.dv; d += 128) {
    const float* src = part_o + (size_t)row * a.dv + d;
    const size_t step = (size_t)n_rows * a.dv;
    float o[4] = {0.f, 0.f, 0.f, 0.f};
    int s = 0;
    for (; s + 4 <= n_splits; s += 4)
#pragma unroll
      for (int u = 0; u < 4; ++u) o[u] = fmaf(src[(s + u) * step], share[s + u], o[u]);
    for (; s < n_splits; ++s) o[0] = fmaf(src[s * step], share[s], o[0]);
    write_gated(g, a, row / a.heads, head, d, (o[0] + o[1]) + (o[2] + o[3]));
  }
}

// ---------------------------------------------------------- simple kernel

// one workgroup of 256 per (token, head): a key per thread for the scores, a
// value dimension per thread for the sum
template <typename T>
__global__ __launch_bounds__(256) void paged_attn_simple(
    const T* __restrict__ q, const T* __restrict__ cache, GatedOut g, PagedRows b, AttnShape a) {
  extern __shared__ float sm[];
  float* qs = sm;                               // [dk]
  float* acc = qs + a.dk;                       // [dv]
  float* p = acc + a.dv;                        // [256]
  long* at = reinterpret_cast<long*>(p + 256);  // [256]
  __shared__ float red[4];
  const int tid = threadIdx.x;
  const int tok = blockIdx.x / a.heads, head = blockIdx.x % a.heads;
  const int kvh = head / (a.heads / a.kv_heads);
  const int seq = b.owner[tok], pos = b.pos[tok];
  const int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  const size_t width = (size_t)a.kv_heads * (a.dk + a.dv);
  const T* keys = cache + (size_t)kvh * a.dk;
  const T* vals = cache + (size_t)a.kv_heads * a.dk + (size_t)kvh * a.dv;
  const float slope = a.slopes ? a.slopes[head] : 0.f;
  for (int d = tid; d < a.dk; d += 256) qs[d] = load_f32(q + (size_t)blockIdx.x * a.dk + d);
  for (int d = tid; d < a.dv; d += 256) acc[d] = 0.f;
  float m = a.sink ? a.sink[head] : NEG_SENTINEL, l = a.sink ? 1.f : 0.f;
  for (int j0 = lo; j0 <= pos; j0 += 256) {
    __syncthreads();
    const int key = j0 + tid;
    float s = NEG_SENTINEL;
    long row = -1;
    if (key <= pos) row = cache_row(b, seq, key);
    if (row >= 0) {
      float dot = 0.f;
      for (int d = 0; d < a.dk; ++d) dot = fmaf(qs[d], load_f32(keys + row * width + d), dot);
      s = dot * a.scale - slope * (float)(pos - key);
    }
    at[tid] = row;
    const float mx = wave_reduce_max(s);
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    const float m_new = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float corr = m <= NEG_THRESHOLD ? 0.f : expf(m - m_new);
    const float e = s <= NEG_THRESHOLD ? 0.f : expf(s - m_new);
    p[tid] = e;
    __syncthreads();  // red is read, p and at are written
    const float sum = wave_reduce_sum(e);
    if ((tid & 63) == 0) red[tid >> 6] = sum;
    __syncthreads();
    l = l * corr + ((red[0] + red[1]) + (red[2] + red[3]));
    m = m_new;
    const int n = min(256, pos - j0 + 1);
    for (int d = tid; d < a.dv; d += 256) {
      float o = acc[d] * corr;
      for (int j = 0; j < n; ++j)
        if (at[j] >= 0) o = fmaf(p[j], load_f32(vals + at[j] * width + d), o);
      acc[d] = o;
    }
  }
  const float inv_l = l > 0.f ? 1.f / l : 0.f;
  for (int d = tid; d < a.dv; d += 256) write_gated(g, a, tok, head, d, acc[d] * inv_l);
}

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

static bool f32_or_bf16(const torch::Tensor& t) {
  TORCH_CHECK(t.is_cuda() && (t.dtype() == torch::kFloat32 || t.dtype() == torch::kBFloat16));
  return t.dtype() == torch::kFloat32;
}

static const float* opt_f32(const c10::optional<torch::Tensor>& t, int64_t n) {
  if (!t.has_value()) return nullptr;
  TORCH_CHECK(t->is_cuda() && t->dtype() == torch::kFloat32 && t->is_contiguous() && t->numel() == n);
  return t->data_ptr<float>();
}

static AttnShape attn_shape(int64_t heads, int64_t kv_heads, int64_t dk, int64_t dv, const torch::Tensor& cache) {
  TORCH_CHECK(kv_heads >= 1 && heads % kv_heads == 0 && dk % 32 == 0 && dv % 16 == 0 && dk > 0 && dv > 0);
  TORCH_CHECK(cache.size(2) == kv_heads * (dk + dv), "cache width mismatch");
  return AttnShape{(int)heads, (int)kv_heads, (int)dk, (int)dv, 0, 1.f, nullptr, nullptr};
}

template <typename K>
static void allow_lds(K kernel, size_t lds) {
  if (lds <= 65536) return;
  TORCH_CHECK(lds <= 160 * 1024, "LDS request of ", lds, " bytes");
  const hipError_t e =
      hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  TORCH_CHECK(e == hipSuccess, "LDS request refused: ", hipGetErrorString(e));
}

template <int RC, int VB>
static void launch_attn(bool decode, dim3 grid, const torch::Tensor& q, const torch::Tensor& cache, GatedOut g,
                        float* po, float* pml, const int* tiles, PagedRows b, AttnShape a, int n_splits) {
  auto stream = at::cuda::getCurrentCUDAStream();
  const int t = q.size(0);
  if (decode) {
    const size_t tile = 4 * (KVT * (VB * 16 + TPAD) + 16 * (KVT + 8)) * 2;
    const size_t merge = (4 * 16 * 2 + 4 * (size_t)(a.heads / a.kv_heads) * a.dv) * 4;
    const size_t lds = std::max(tile, merge);
    allow_lds(&paged_attn_decode<RC, VB>, lds);
    paged_attn_decode<RC, VB><<<grid, 256, lds, stream>>>(BF16P(q), BF16P(cache), g, po, pml, b, a, t, n_splits);
  } else {
    const size_t lds = (2 * KVT * (RC * 32 + VB * 16 + 2 * TPAD) + 4 * 16 * (KVT + 8)) * 2;
    allow_lds(&paged_attn_kernel<RC, VB>, lds);
    paged_attn_kernel<RC, VB><<<grid, 256, lds, stream>>>(BF16P(q), BF16P(cache), g, po, pml, tiles, b, a, t, n_splits);
  }
}

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
  const bool f32 = f32_or_bf16(q);
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous() && q.dtype() == cache.dtype());
  const int t = q.size(0), heads = q.size(1), dk = q.size(2);
  const PagedRows b = paged_rows(pos, owner, tables, cache, t);
  AttnShape a = attn_shape(heads, kv_heads, dk, dv, cache);
  a.window = window;
  a.scale = scale;
  a.slopes = opt_f32(slopes, heads);
  a.sink = opt_f32(sink, heads);
  auto out = torch::empty({t, (long)heads * dv}, q.options().dtype(out_f32 ? torch::kFloat32 : torch::kBFloat16));
  if (t == 0) return out;
  GatedOut g{out.data_ptr(), nullptr, 0, out_f32};
  if (gate.has_value()) {
    TORCH_CHECK(gate->is_cuda() && gate->dim() == 2 && gate->stride(1) == 1 && gate->dtype() == out.dtype());
    TORCH_CHECK(gate->size(0) == t && gate->size(1) == (long)heads * dv);
    g.gate = gate->data_ptr();
    g.gate_stride = gate->stride(0);
  }
  auto stream = at::cuda::getCurrentCUDAStream();
  if (f32 || dk > 256 || dv > 256) {
    const size_t lds = ((size_t)dk + dv + 256) * 4 + 256 * 8;
    TORCH_CHECK(lds <= 65536, "head sizes ", dk, " and ", dv, " are not supported");
    if (f32) {
      paged_attn_simple<float><<<t * heads, 256, lds, stream>>>(q.data_ptr<float>(), cache.data_ptr<float>(), g, b, a);
    } else {
      paged_attn_simple<unsigned short><<<t * heads, 256, lds, stream>>>(BF16P(q), BF16P(cache), g, b, a);
    }
    HIP_CHECK_LAST();
    return out;
  }
  TORCH_CHECK(splits <= 64 && run_tokens >= 1, "at most 64 key splits");
  TORCH_CHECK(tiles.is_cuda() && tiles.dtype() == torch::kInt32 && tiles.is_contiguous() && tiles.dim() == 2);
  const int group = heads / (int)kv_heads;
  const bool decode = run_tokens == 1 && group <= 16 && tiles.size(0) == t;
  const int row_groups = ((int)run_tokens * group + 63) / 64;
  dim3 grid(tiles.size(0), kv_heads * (decode ? 1 : row_groups), 1);
  int n_splits = (int)splits;
  if (n_splits <= 0) {
    // enough workgroups for the chip; a decoding workgroup reads 4 tiles at once
    const long tiles_per = decode ? 4 : 1, wanted = decode ? 512 : 256;
    const long wgs = (long)grid.x * grid.y;
    n_splits = (int)std::max(
        1L, std::min({(long)((max_keys + KVT * tiles_per - 1) / (KVT * tiles_per)), wanted / std::max(1L, wgs), 64L}));
  }
  grid.z = n_splits;
  auto f32o = q.options().dtype(torch::kFloat32);
  auto part_o = torch::empty({n_splits > 1 ? (long)n_splits * t * heads * dv : 0}, f32o);
  auto part_ml = torch::empty({n_splits > 1 ? (long)n_splits * t * heads * 2 : 0}, f32o);
  float* po = n_splits > 1 ? part_o.data_ptr<float>() : nullptr;
  float* pml = n_splits > 1 ? part_ml.data_ptr<float>() : nullptr;
#define PA(RC, VB) launch_attn<RC, VB>(decode, grid, q, cache, g, po, pml, tiles.data_ptr<int>(), b, a, n_splits)
#define PAV(RC)            \
  do {                     \
    if (dv <= 32) PA(RC, 2); \
    else if (dv <= 64) PA(RC, 4); \
    else if (dv <= 128) PA(RC, 8); \
    else PA(RC, 16);       \
  } while (0)
  if (dk <= 32) PAV(1);
  else if (dk <= 64) PAV(2);
  else if (dk <= 128) PAV(4);
  else PAV(8);
#undef PAV
#undef PA
  HIP_CHECK_LAST();
  if (n_splits > 1) {
    paged_attn_combine<<<t * heads, 128, 0, stream>>>(po, pml, g, a, t * heads, n_splits);
    HIP_CHECK_LAST();
  }
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
  const AttnShape a = attn_shape(heads, kv_heads, dk, dv, cache);
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
