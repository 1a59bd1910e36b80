// Attention over paged keys and values for CDNA4 (gfx950), shared by the kinds of
// attention that are compiled from it (paged_attn.hip, capped_attn.hip,
// sigmoid_attn.hip, paired_attn.hip): grouped heads with separate key and value sizes,
// and as arguments a sliding window or chunks, a bias per head that grows with the
// distance, one learned entry of the softmax's denominator per head (a sink), and a
// sigmoid gate on the output. What differs inside the loops is a template argument:
//
//   KIND   how scores become weights: a softmax, a softmax of scores capped by a tanh,
//          or a sigmoid of every score for itself
//   MAPS   weights per head. 2: both mix the same values, and the head's result is
//          N(o_1 - share o_2) factor, N dividing by the root mean square
//
// A token's cache row is [G heads of MAPS x DK keys | G heads of DV values], DK a
// multiple of 32 and DV of 16 (padded with zeros when weights are packed).
//
//   paged_attn_kernel   MFMA flash kernel for prompts and portions: 4 waves of 16 or 32
//                       (token, head) rows share double-buffered key/value tiles
//   paged_attn_decode   few rows per kv head: every wave takes tiles of its own,
//                       keys straight from memory, merged through LDS at the end
//   paged_attn_combine  merges key splits
//   paged_attn_simple   any size, 32-bit or bf16 storage
//
// Every page index is checked against the pool before it is used.
#pragma once

#include "common.h"
#include "paged.h"
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>
#include <algorithm>

#define KVT 32   // keys per tile of a decoding wave; tiles are aligned, so one lies in one page
#define TPAD 16  // LDS row padding (elements)
#define LOG2E 1.4426950408889634f

enum ScoreKind : int { SOFTMAX = 0, CAPPED = 1, SIGMOID = 2 };

struct AttnShape {
  int heads, kv_heads, dk, dv;  // padded head sizes
  int window;                   // 0: everything before
  int chunk;                    // 0: no chunks; else a row sees its own run of this many positions
  float scale;
  const float* slopes;  // SOFTMAX: [heads] or null
  const float* sink;    // SOFTMAX, CAPPED: [heads] or null
  const float* bias;    // SIGMOID: [heads], added to the scores
  float cap;            // CAPPED: cap * tanh(score / cap)
  float share, factor, eps;  // MAPS == 2
  int vdim;                  // MAPS == 2: size of a head without padding
};

// the first key that position pos sees (may be negative)
__device__ __forceinline__ int first_key(const AttnShape& a, int pos) {
  return a.window > 0 ? pos - a.window + 1 : a.chunk > 0 ? pos - pos % a.chunk : 0;
}

// where the result goes: out[t, head * dv + c] = o * sigmoid(gate), gate[t, head * dv + c] or gate[t, head]
struct GatedOut {
  void* out;         // row stride out_stride
  long out_stride;
  const void* gate;  // row stride gate_stride, or null
  long gate_stride;
  bool per_head;     // one gate per head
  bool f32;          // both in 32-bit, else bf16
  bool by4;          // groups of 4 of the result are aligned
};

__device__ __forceinline__ float gate_of(const GatedOut& g, size_t at) {
  const float z = g.f32 ? reinterpret_cast<const float*>(g.gate)[at]
                        : bf16_to_f32(reinterpret_cast<const unsigned short*>(g.gate)[at]);
  return 1.f / (1.f + expf(-z));
}

__device__ __forceinline__ void write_gated(const GatedOut& g, const AttnShape& a, size_t tok, int head, int c, float v) {
  const int col = head * a.dv + c;
  if (g.gate) v *= gate_of(g, tok * g.gate_stride + (g.per_head ? head : col));
  const size_t to = tok * g.out_stride + col;
  if (g.f32) reinterpret_cast<float*>(g.out)[to] = v;
  else reinterpret_cast<unsigned short*>(g.out)[to] = f32_to_bf16(v);
}

// 4 neighbouring values, c a multiple of 4
__device__ __forceinline__ void write_gated4(const GatedOut& g, const AttnShape& a, size_t tok, int head, int c, f32x4 v) {
  const int col = head * a.dv + c;
  if (g.gate) {
    const size_t at = tok * g.gate_stride + (g.per_head ? head : col);
    if (g.per_head) {
      v *= gate_of(g, at);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] *= gate_of(g, at + e);
    }
  }
  const size_t to = tok * g.out_stride + col;
  if (!g.by4) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      if (g.f32) reinterpret_cast<float*>(g.out)[to + e] = v[e];
      else reinterpret_cast<unsigned short*>(g.out)[to + e] = f32_to_bf16(v[e]);
    }
  } else if (g.f32) {
    *reinterpret_cast<f32x4*>(reinterpret_cast<float*>(g.out) + to) = v;
  } else {
    *reinterpret_cast<v4s*>(reinterpret_cast<unsigned short*>(g.out) + to) =
        v4s{(short)f32_to_bf16(v[0]), (short)f32_to_bf16(v[1]), (short)f32_to_bf16(v[2]), (short)f32_to_bf16(v[3])};
  }
}

__device__ __forceinline__ void wave_lds_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// A tile's scores are computed as K Q^T and its result as V^T P^T: a lane then holds
// keys (or value dimensions) of ONE query row, the row of its column lane&15, so that a
// softmax's maximum and sum take two exchanges between lanes, and the weights are the
// next product's operand as they are. In the C layout, register r of block nb is key
// nb*16 + hi*4 + r; as operand of a product over 32 keys, registers 0-3 of two blocks
// are its 8 elements, so the values are read in the same order (load_values).

// factors of a raw score, in log2 units
struct ScoreScale {
  float in;      // SOFTMAX, SIGMOID: scale; CAPPED: 2 scale / cap
  float cap;     // CAPPED
  bool bounded;  // weights need no maximum: the cap keeps them and their sums in range
};

template <int KIND>
__device__ __forceinline__ ScoreScale score_scale(const AttnShape& a) {
  if (KIND == CAPPED) return ScoreScale{2.f * a.scale / a.cap * LOG2E, a.cap * LOG2E, a.cap * LOG2E <= 80.f};
  return ScoreScale{a.scale * LOG2E, 0.f, KIND == SIGMOID};
}

__device__ __forceinline__ float first_maximum(const ScoreScale& k) { return k.bounded ? 0.f : NEG_SENTINEL; }

// the keys that a lane's query row sees: [lo, pos], none if pos < 0
struct SeenRow {
  int pos, lo;
};

// in log2 units: SOFTMAX: slope per distance; SIGMOID: bias
template <int KIND>
__device__ __forceinline__ float linear_term(const AttnShape& a, int head) {
  if (KIND == SOFTMAX) return a.slopes ? a.slopes[head] * LOG2E : 0.f;
  return KIND == SIGMOID && a.bias ? a.bias[head] * LOG2E : 0.f;
}

// maximum and sum over the lanes of a query row
__device__ __forceinline__ float row_max(float x) {
  x = fmaxf(x, __shfl_xor(x, 16, WAVE));
  return fmaxf(x, __shfl_xor(x, 32, WAVE));
}
__device__ __forceinline__ float row_sum(float x) {
  x += __shfl_xor(x, 16, WAVE);
  return x + __shfl_xor(x, 32, WAVE);
}

// Scores of a lane's row and NB blocks of 16 keys from j0 -> weights, in place.
// m: the row's maximum so far; l: this lane's share of the sum. Returns whether m grew
// in some row of the wave; what has been summed is then to be scaled by corr.
template <int KIND, int NB>
__device__ __forceinline__ bool weigh_tile(
    f32x4* s, float& m, float& l, float lin, SeenRow n, int j0, int hi, int j_end, bool interior, ScoreScale k,
    float& corr) {
  const int first = j0 + hi * 4;  // key of register 0 in block 0
  if (KIND == SIGMOID) {
#pragma unroll
    for (int nb = 0; nb < NB; ++nb)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        s[nb][r] = __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(fminf(fmaf(s[nb][r], -k.in, -lin), 100.f)));
    if (!interior) {
#pragma unroll
      for (int nb = 0; nb < NB; ++nb)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int key = first + nb * 16 + r;
          if (key >= j_end || key > n.pos || key < n.lo) s[nb][r] = 0.f;
        }
    }
    return false;
  }
  const float base = KIND == SOFTMAX ? lin * (float)(n.pos - first) : 0.f;
#pragma unroll
  for (int nb = 0; nb < NB; ++nb)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if (KIND == SOFTMAX) {
        s[nb][r] = fmaf(s[nb][r], k.in, fmaf(lin, (float)(nb * 16 + r), -base));
      } else {  // tanh(x) = 1 - 2 / (exp(2x) + 1)
        const float e = __builtin_amdgcn_exp2f(fminf(s[nb][r] * k.in, 80.f));
        s[nb][r] = fmaf(-2.f * k.cap, __builtin_amdgcn_rcpf(e + 1.f), k.cap);
      }
    }
  // masking and the maximum stay in separate loops (see prefill_attn.hip)
  if (!interior) {
#pragma unroll
    for (int nb = 0; nb < NB; ++nb)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = first + nb * 16 + r;
        if (key >= j_end || key > n.pos || key < n.lo) s[nb][r] = NEG_SENTINEL;
      }
  }
  bool grew = false;
  corr = 1.f;
  if (KIND != CAPPED || !k.bounded) {
    float mx = m;
#pragma unroll
    for (int nb = 0; nb < NB; ++nb)
#pragma unroll
      for (int r = 0; r < 4; ++r) mx = fmaxf(mx, s[nb][r]);
    const float m_new = row_max(mx);
    grew = __any(m_new > m);
    if (grew) {
      corr = m <= NEG_THRESHOLD ? 0.f : exp2f(m - m_new);
      l *= corr;
      m = m_new;
    }
  }
  const float top = m <= NEG_THRESHOLD ? 0.f : m;  // nothing seen yet: weights of 0
  float sum = 0.f;
#pragma unroll
  for (int nb = 0; nb < NB; ++nb)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      s[nb][r] = __builtin_amdgcn_exp2f(s[nb][r] - top);
      sum += s[nb][r];
    }
  l += sum;
  return grew;
}

// weights of 32 keys as an operand
__device__ __forceinline__ bf16x8 weight_operand(const f32x4& a, const f32x4& b) {
  using f32x8 = __attribute__((ext_vector_type(8))) float;
  using nbf16x8 = __attribute__((ext_vector_type(8))) __bf16;
  const f32x8 v = {a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
  return __builtin_bit_cast(bf16x8, __builtin_convertvector(v, nbf16x8));
}

// Values of one dimension per lane (column lane&15 of a block) in the order of
// weight_operand, by two transposing LDS loads. p: row hi*4 + (lane&15)/4, column
// 4*(lane&3) of the block, in the tile's rows of these 32 keys.
__device__ __forceinline__ bf16x8 load_values(const unsigned short* p, int row_elems) {
  using lds_v4s = __attribute__((address_space(3))) v4s;
  const v4s a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s*)p);
  const v4s b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s*)(p + 16 * row_elems));
  return bf16x8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}

// ------------------------------------------------------------ MFMA kernel

// The token run (x) and the heads (y) of a workgroup. Workgroups are dealt to the 8
// chiplets in turn: each chiplet takes heads of its own, whose keys and values then stay
// in its cache. Late rows see most and come first; every second 32 are turned round, so
// that a compute unit (there are 32 on a chiplet) that gets two gets a long and a short one.
__device__ __forceinline__ int2 spread_tiles(int nx, int ny) {
  unsigned at = blockIdx.y * nx + blockIdx.x;
  if (ny % 8 == 0) {
    const unsigned per = ny / 8;
    unsigned i = at / 8;
    if (i / 32 * 32 + 32 <= nx * per && (i & 32)) i = i / 32 * 32 + 31 - i % 32;
    return int2{(int)(nx - 1 - i / per), (int)((at & 7) * per + i % per)};
  }
  if (nx * ny % 8 == 0) at = (at & 7) * (nx * ny / 8) + at / 8;
  return int2{(int)(nx - 1 - at % nx), (int)(at / nx)};
}

// RC: 32-wide chunks of the key size, VB: 16-wide blocks of the value size, at
// least as many as there are: tiles are filled up with zeros, so that no branch
// stands between products. A wave holds all maps of its QB blocks of 16 rows; a tile
// has KT keys and lies in one page.
// Grid: (token runs, kv heads x groups of 64 QB rows, key splits).
template <int KIND, int MAPS, int RC, int VB, int QB, int KT>
__global__ __launch_bounds__(256, QB) void paged_attn_kernel(
    const unsigned short* __restrict__ q,      // [T, H, MAPS, dk]
    const unsigned short* __restrict__ cache,  // [pages, PAGE, G * (MAPS * dk + dv)]
    GatedOut g,                                // n_splits == 1
    float* __restrict__ part_o,                // [n_splits, T*H, MAPS, dv]
    float* __restrict__ part_ml,               // [n_splits, T*H, MAPS, 2]
    const int* __restrict__ tiles,             // [n, 2] first token, token count
    PagedRows b, AttnShape a, int total_tokens, int n_splits) {
  constexpr int ROWS = 64 * QB, NB = KT / 16;
  constexpr int KROW = MAPS * RC * 32 + TPAD, VROW = VB * 16 + TPAD;
  constexpr int K8 = MAPS * RC * 4, V8 = VB * 2;             // 16-byte groups of a row
  constexpr int K_LOADS = KT * K8, LOADS = KT * (K8 + V8);
  constexpr int NLD = (LOADS + 255) / 256;                   // per thread
  const int2 own = spread_tiles(gridDim.x, gridDim.y);
  const int bx = own.x, by = own.y;
  const int tok0 = tiles[2 * bx];
  const int ntok = tiles[2 * bx + 1];
  const int group = a.heads / a.kv_heads;
  const int rows = ntok * group;
  const int kvh = by % a.kv_heads;
  const int g0 = by / a.kv_heads * ROWS;
  if (g0 >= rows) return;  // uniform over the workgroup
  const int g1 = min(g0 + ROWS, rows);

  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & (WAVE - 1);
  const int col = lane & 15, hi = lane >> 4;
  const int r0 = g0 + wave * 16 * QB;

  extern __shared__ unsigned short smem[];

  const int seq = b.owner[tok0];
  const int first_pos = b.pos[tok0 + g0 / group];
  const int last_pos = b.pos[tok0 + (g1 - 1) / group];
  const int key_lo = max(0, first_key(a, first_pos)) / KT * KT;
  const int key_hi = last_pos + 1;
  const int n_tiles = (key_hi - key_lo + KT - 1) / KT;
  const int per_split = (n_tiles + n_splits - 1) / n_splits;
  const int j_begin = key_lo + blockIdx.z * per_split * KT;
  const int j_end = min(key_hi, j_begin + per_split * KT);

  const ScoreScale scale = score_scale<KIND>(a);
  bf16x8 q_frag[QB][MAPS][RC];
  f32x4 acc_o[QB][MAPS][VB];
  float m[QB][MAPS], l[QB][MAPS], lin[QB];
  SeenRow seen[QB];
#pragma unroll
  for (int i = 0; i < QB; ++i) {
    const int row = r0 + i * 16 + col;
    const bool live = row < rows;
    const int head = live ? kvh * group + row % group : 0;
    const size_t at = ((size_t)(tok0 + (live ? row / group : 0)) * a.heads + head) * MAPS * a.dk;
    seen[i].pos = live ? b.pos[tok0 + row / group] : -1;  // -1: sees nothing
    seen[i].lo = live ? first_key(a, seen[i].pos) : 0;
    lin[i] = live ? linear_term<KIND>(a, head) : 0.f;
#pragma unroll
    for (int u = 0; u < MAPS; ++u) {
      m[i][u] = first_maximum(scale);
      l[i][u] = 0.f;
#pragma unroll
      for (int kc = 0; kc < RC; ++kc)
        q_frag[i][u][kc] = live && kc * 32 < a.dk
                               ? *reinterpret_cast<const bf16x8*>(q + at + u * a.dk + kc * 32 + hi * 8)
                               : bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
      for (int d = 0; d < VB; ++d) acc_o[i][u][d] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
  }
  // keys that every row of this wave sees: [all_lo, all_hi]; those that some row sees: [any_lo, any_hi]
  const bool full_wave = r0 + 16 * QB <= rows;
  const int wave_first = r0 < rows ? b.pos[tok0 + r0 / group] : -1;
  const int wave_last = r0 < rows ? b.pos[tok0 + (min(r0 + 16 * QB, rows) - 1) / group] : -1;
  const int all_hi = full_wave ? wave_first : -1;
  const int all_lo = full_wave ? first_key(a, wave_last) : 0;
  const int any_hi = wave_last, any_lo = r0 < rows ? first_key(a, wave_first) : 0;

  const int width = a.kv_heads * (MAPS * a.dk + a.dv);
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
        const int u = is_v ? 0 : idx % K8 / (RC * 4);
        const int c8 = (is_v ? (idx - K_LOADS) % V8 : idx % (RC * 4)) * 8;
        const int c = is_v ? a.kv_heads * MAPS * a.dk + kvh * a.dv + c8 : (kvh * MAPS + u) * a.dk + c8;
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
        unsigned short* dst = is_v ? buf + KT * KROW + row * VROW + c8 : buf + row * KROW + c8;
        *reinterpret_cast<bf16x8*>(dst) = next[i];
      }
    }
  };

  if (j_begin < j_end) {
    fetch(j_begin);
    stage(smem);
  }
  __syncthreads();
  int which = 0;
  for (int j0 = j_begin; j0 < j_end; j0 += KT, which ^= 1) {
    const unsigned short* k_lds = smem + which * KT * (KROW + VROW);
    const bool more = j0 + KT < j_end;
    if (more) fetch(j0 + KT);
    if (j0 <= any_hi && j0 + KT > any_lo) {  // uniform over the wave
      const bool interior = j0 >= all_lo && j0 + KT - 1 <= all_hi && j0 + KT <= j_end;
      bf16x8 p_frag[QB][MAPS][NB / 2];
#pragma unroll
      for (int u = 0; u < MAPS; ++u) {
        f32x4 s[QB][NB];
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) {
#pragma unroll
          for (int i = 0; i < QB; ++i) s[i][nb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int kc = 0; kc < RC; ++kc) {
            const bf16x8 kt =
                *reinterpret_cast<const bf16x8*>(&k_lds[(nb * 16 + col) * KROW + (u * RC + kc) * 32 + hi * 8]);
#pragma unroll
            for (int i = 0; i < QB; ++i)
              s[i][nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kt, q_frag[i][u][kc], s[i][nb], 0, 0, 0);
          }
        }
#pragma unroll
        for (int i = 0; i < QB; ++i) {
          float corr;
          if (weigh_tile<KIND, NB>(s[i], m[i][u], l[i][u], lin[i], seen[i], j0, hi, j_end, interior, scale, corr)) {
#pragma unroll
            for (int d = 0; d < VB; ++d) acc_o[i][u][d] *= corr;
          }
#pragma unroll
          for (int ks = 0; ks < NB / 2; ++ks) p_frag[i][u][ks] = weight_operand(s[i][2 * ks], s[i][2 * ks + 1]);
        }
      }
      const unsigned short* v_lds = k_lds + KT * KROW + (hi * 4 + col / 4) * VROW + (col & 3) * 4;
#pragma unroll
      for (int d = 0; d < VB; ++d)
#pragma unroll
        for (int ks = 0; ks < NB / 2; ++ks) {
          const bf16x8 vt = load_values(v_lds + ks * 32 * VROW + d * 16, VROW);
#pragma unroll
          for (int i = 0; i < QB; ++i)
#pragma unroll
            for (int u = 0; u < MAPS; ++u)
              acc_o[i][u][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, p_frag[i][u][ks], acc_o[i][u][d], 0, 0, 0);
        }
    }
    if (more) stage(smem + (which ^ 1) * KT * (KROW + VROW));
    __syncthreads();
  }

#pragma unroll
  for (int i = 0; i < QB; ++i) {
    const int row = r0 + i * 16 + col;
    const bool live = row < rows;
    const size_t tok = tok0 + (live ? row / group : 0);
    const int head = kvh * group + (live ? row % group : 0);
    float inv[MAPS];
#pragma unroll
    for (int u = 0; u < MAPS; ++u) inv[u] = KIND == SIGMOID ? 1.f : row_sum(l[i][u]);
    if (n_splits > 1) {
      if (!live) continue;
      const size_t at = (((size_t)blockIdx.z * total_tokens + tok) * a.heads + head) * MAPS;
#pragma unroll
      for (int u = 0; u < MAPS; ++u) {
#pragma unroll
        for (int d = 0; d < VB; ++d)
          if (d * 16 < a.dv) *reinterpret_cast<f32x4*>(part_o + (at + u) * a.dv + d * 16 + hi * 4) = acc_o[i][u][d];
        if (KIND != SIGMOID && hi == 0) {
          part_ml[(at + u) * 2] = m[i][u];
          part_ml[(at + u) * 2 + 1] = inv[u];
        }
      }
      continue;
    }
    if (KIND != SIGMOID) {
#pragma unroll
      for (int u = 0; u < MAPS; ++u) {
        float up = 1.f, sum = inv[u];
        if (a.sink) {
          const float z = a.sink[head] * LOG2E, top = fmaxf(m[i][u], z);
          up = exp2f(m[i][u] - top);
          sum = sum * up + exp2f(z - top);
        }
        inv[u] = sum > 0.f ? up / sum : 0.f;
      }
    }
    if (MAPS == 2) {
      float ss = 0.f;
#pragma unroll
      for (int d = 0; d < VB; ++d)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float o = acc_o[i][0][d][r] * inv[0] - a.share * (acc_o[i][MAPS - 1][d][r] * inv[MAPS - 1]);
          acc_o[i][0][d][r] = o;
          ss = fmaf(o, o, ss);  // padding is zero
        }
      inv[0] = a.factor / sqrtf(row_sum(ss) / a.vdim + a.eps);
    }
    if (!live) continue;
#pragma unroll
    for (int d = 0; d < VB; ++d)
      if (d * 16 < a.dv) write_gated4(g, a, tok, head, d * 16 + hi * 4, acc_o[i][0][d] * inv[0]);
  }
}

// --------------------------------------------------------------- few rows

// One token and one kv head with at most 16 query heads. Grid: (tokens, kv
// heads, key splits); the 4 waves of a workgroup take every fourth tile. Two maps
// always leave their parts to the combining kernel.
template <int KIND, int MAPS, int RC, int VB>
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
  unsigned short* v_tile = smem + wave * KVT * VROW;

  const int seq = b.owner[tok], pos = b.pos[tok];
  const int lo = first_key(a, pos), key_lo = max(0, lo) / KVT * KVT;
  const int n_tiles = (pos + 1 - key_lo + KVT - 1) / KVT;
  const int per_split = (n_tiles + n_splits - 1) / n_splits;
  const int j_begin = key_lo + blockIdx.z * per_split * KVT;
  const int j_end = min(pos + 1, j_begin + per_split * KVT);

  const ScoreScale scale = score_scale<KIND>(a);
  const bool live = col < group;
  const SeenRow seen{live ? pos : -1, lo};
  const float lin = live ? linear_term<KIND>(a, kvh * group + col) : 0.f;
  bf16x8 q_frag[MAPS][RC];
  f32x4 acc_o[MAPS][VB];
  float m[MAPS], l[MAPS];
  const size_t q_at = ((size_t)tok * a.heads + kvh * group + col) * MAPS * a.dk;
#pragma unroll
  for (int u = 0; u < MAPS; ++u) {
    m[u] = first_maximum(scale);
    l[u] = 0.f;
#pragma unroll
    for (int kc = 0; kc < RC; ++kc)
      q_frag[u][kc] = live && kc * 32 < a.dk
                          ? *reinterpret_cast<const bf16x8*>(q + q_at + u * a.dk + kc * 32 + hi * 8)
                          : bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
    for (int d = 0; d < VB; ++d) acc_o[u][d] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const int width = a.kv_heads * (MAPS * a.dk + a.dv);
  for (int j0 = j_begin + wave * KVT; j0 < j_end; j0 += 4 * KVT) {
    const long at = cache_row(b, seq, j0);
    bf16x8 vals[NLD], kt[MAPS][2][RC];
#pragma unroll
    for (int u = 0; u < MAPS; ++u)
#pragma unroll
      for (int nb = 0; nb < 2; ++nb)
#pragma unroll
        for (int kc = 0; kc < RC; ++kc) {
          const int row = nb * 16 + col;
          kt[u][nb][kc] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
          if (kc * 32 < a.dk && at >= 0 && j0 + row < j_end)
            kt[u][nb][kc] = *reinterpret_cast<const bf16x8*>(
                cache + ((size_t)at + row) * width + (kvh * MAPS + u) * a.dk + kc * 32 + hi * 8);
        }
#pragma unroll
    for (int i = 0; i < NLD; ++i) {
      const int idx = lane + i * WAVE, row = idx / V8, c8 = idx % V8 * 8;
      vals[i] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
      if (at >= 0 && j0 + row < j_end && c8 < a.dv)
        vals[i] = *reinterpret_cast<const bf16x8*>(
            cache + ((size_t)at + row) * width + a.kv_heads * MAPS * a.dk + kvh * a.dv + c8);
    }
    bf16x8 p_frag[MAPS];
#pragma unroll
    for (int u = 0; u < MAPS; ++u) {
      f32x4 s[2];
#pragma unroll
      for (int nb = 0; nb < 2; ++nb) {
        s[nb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kc = 0; kc < RC; ++kc)
          s[nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kt[u][nb][kc], q_frag[u][kc], s[nb], 0, 0, 0);
      }
      float corr;
      if (weigh_tile<KIND, 2>(s, m[u], l[u], lin, seen, j0, hi, j_end, false, scale, corr)) {
#pragma unroll
        for (int d = 0; d < VB; ++d) acc_o[u][d] *= corr;
      }
      p_frag[u] = weight_operand(s[0], s[1]);
    }
    wave_lds_fence();  // the last tile's reads are done
#pragma unroll
    for (int i = 0; i < NLD; ++i) {
      const int idx = lane + i * WAVE, row = idx / V8, c8 = idx % V8 * 8;
      *reinterpret_cast<bf16x8*>(&v_tile[row * VROW + c8]) = vals[i];
    }
    wave_lds_fence();
    const unsigned short* v_lds = v_tile + (hi * 4 + col / 4) * VROW + (col & 3) * 4;
#pragma unroll
    for (int d = 0; d < VB; ++d) {
      const bf16x8 vt = load_values(v_lds + d * 16, VROW);
#pragma unroll
      for (int u = 0; u < MAPS; ++u)
        acc_o[u][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, p_frag[u], acc_o[u][d], 0, 0, 0);
    }
  }
  // merge the waves: [MAPS][4][16] maxima and sums, then [MAPS][4][group][dv] weighted sums
  __syncthreads();
  float* ml = reinterpret_cast<float*>(smem);   // [MAPS][4][16][2]
  float* os = ml + MAPS * 4 * 16 * 2;           // [MAPS][4][group][dv]
#pragma unroll
  for (int u = 0; u < MAPS; ++u) {
    const float sum = KIND == SIGMOID ? 1.f : row_sum(l[u]);
    if (!live) continue;
    if (hi == 0) {
      ml[((u * 4 + wave) * 16 + col) * 2] = m[u];
      ml[((u * 4 + wave) * 16 + col) * 2 + 1] = sum;
    }
#pragma unroll
    for (int d = 0; d < VB; ++d)
      if (d * 16 < a.dv)
        *reinterpret_cast<f32x4*>(os + ((u * 4 + wave) * group + col) * a.dv + d * 16 + hi * 4) = acc_o[u][d];
  }
  __syncthreads();
  for (int i = tid; i < MAPS * group * a.dv; i += 256) {
    const int u = MAPS == 1 ? 0 : i / (group * a.dv), in = i - u * group * a.dv;
    const int row = in / a.dv, c = in - row * a.dv, head = kvh * group + row;
    const float* mlu = ml + u * 4 * 16 * 2;
    const float* osu = os + u * 4 * group * a.dv;
    float sum = 0.f, o = 0.f, top = 0.f;
    if (KIND == SIGMOID) {
#pragma unroll
      for (int v = 0; v < 4; ++v) o += osu[(v * group + row) * a.dv + c];
    } else {
      top = NEG_SENTINEL;
#pragma unroll
      for (int v = 0; v < 4; ++v) top = fmaxf(top, mlu[(v * 16 + row) * 2]);
    }
    const float own = top;
    if (KIND != SIGMOID) {
      if (MAPS == 1 && n_splits == 1 && a.sink) top = fmaxf(top, a.sink[head] * LOG2E);
#pragma unroll
      for (int v = 0; v < 4; ++v) {
        const float mv = mlu[(v * 16 + row) * 2];
        const float e = mv > NEG_THRESHOLD ? exp2f(mv - top) : 0.f;
        sum = fmaf(e, mlu[(v * 16 + row) * 2 + 1], sum);
        o = fmaf(e, osu[(v * group + row) * a.dv + c], o);
      }
    }
    if (MAPS == 1 && n_splits == 1) {
      if (KIND != SIGMOID) {
        if (a.sink) sum += exp2f(a.sink[head] * LOG2E - top);
        o = sum > 0.f ? o / sum : 0.f;
      }
      write_gated(g, a, tok, head, c, o);
    } else {
      const size_t at = (((size_t)blockIdx.z * total_tokens + tok) * a.heads + head) * MAPS + u;
      part_o[at * a.dv + c] = o;
      if (KIND != SIGMOID && c == 0) {
        part_ml[at * 2] = own;
        part_ml[at * 2 + 1] = sum;
      }
    }
  }
}

#define COMBINE_THREADS(MAPS) ((MAPS) == 1 ? 128 : 512)

// one workgroup per (token, head) row; two maps (dv <= 256): half of the threads for each
template <int KIND, int MAPS>
__global__ __launch_bounds__(COMBINE_THREADS(MAPS)) void paged_attn_combine(
    const float* __restrict__ part_o, const float* __restrict__ part_ml, GatedOut g, AttnShape a, int n_rows,
    int n_splits) {
  __shared__ float share[MAPS][WAVE];  // weight of each split in the row
  const int row = blockIdx.x, head = row % a.heads, tid = threadIdx.x;
  if (KIND == SIGMOID) {
    if (tid < WAVE) share[0][tid] = 1.f;
  } else if (tid < MAPS * WAVE) {  // a wave for each map
    const int s = tid & (WAVE - 1), u = tid / WAVE;
    float m = NEG_SENTINEL, l = 0.f;
    if (s < n_splits) {
      const size_t at = (((size_t)s * n_rows + row) * MAPS + u) * 2;
      m = part_ml[at];
      l = part_ml[at + 1];
    }
    float mx = wave_reduce_max(m);
    if (a.sink) mx = fmaxf(mx, a.sink[head] * LOG2E);
    const float w = m > NEG_THRESHOLD ? exp2f(m - mx) : 0.f;
    float sum = wave_reduce_sum(w * l);
    if (a.sink) sum += exp2f(a.sink[head] * LOG2E - mx);
    share[u][s] = sum > 0.f ? w / sum : 0.f;
  }
  __syncthreads();
  const size_t step = (size_t)n_rows * MAPS * a.dv;
  auto summed = [&](int u, int d) {
    const float* src = part_o + ((size_t)row * MAPS + u) * a.dv + d;
    float o[4] = {0.f, 0.f, 0.f, 0.f};
    int s = 0;
    for (; s + 4 <= n_splits; s += 4)
#pragma unroll
      for (int v = 0; v < 4; ++v) o[v] = fmaf(src[(s + v) * step], share[u][s + v], o[v]);
    for (; s < n_splits; ++s) o[0] = fmaf(src[s * step], share[u][s], o[0]);
    return (o[0] + o[1]) + (o[2] + o[3]);
  };
  if (MAPS == 1) {
    for (int d = tid; d < a.dv; d += 128) write_gated(g, a, row / a.heads, head, d, summed(0, d));
    return;
  }
  __shared__ float second[256], red[4];
  const int d = tid & 255;
  float o = d < a.dv ? summed(tid / 256, d) : 0.f;
  if (tid >= 256) second[d] = o;
  __syncthreads();
  if (tid < 256) {
    o -= a.share * second[d];
    const float ss = wave_reduce_sum(o * o);
    if ((tid & (WAVE - 1)) == 0) red[tid / WAVE] = ss;
  }
  __syncthreads();
  if (d >= a.dv || tid >= 256) return;
  const float inv = a.factor / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / a.vdim + a.eps);
  write_gated(g, a, row / a.heads, head, d, o * inv);
}

// ---------------------------------------------------------- simple kernel

// one workgroup of 256 per (token, head): a key per thread for the scores, a
// value dimension per thread for the sum; one map after the other
template <int KIND, int MAPS, typename T>
__global__ __launch_bounds__(256) void paged_attn_simple(
    const T* __restrict__ q, const T* __restrict__ cache, GatedOut g, PagedRows b, AttnShape a) {
  extern __shared__ float sm[];
  float* p = sm;                                // [256]
  long* at = reinterpret_cast<long*>(p + 256);  // [256]
  float* qs = reinterpret_cast<float*>(at + 256);  // [dk]
  float* acc0 = qs + a.dk;                      // [MAPS][dv]
  __shared__ float red[4];
  const int tid = threadIdx.x;
  const int tok = blockIdx.x / a.heads, head = blockIdx.x % a.heads;
  const int kvh = head / (a.heads / a.kv_heads);
  const int seq = b.owner[tok], pos = b.pos[tok];
  const int lo = max(0, first_key(a, pos));
  const size_t width = (size_t)a.kv_heads * (MAPS * a.dk + a.dv);
  const T* vals = cache + (size_t)a.kv_heads * MAPS * a.dk + (size_t)kvh * a.dv;
  const float slope = KIND == SOFTMAX && a.slopes ? a.slopes[head] : 0.f;
  const float bias = KIND == SIGMOID && a.bias ? a.bias[head] : 0.f;
  for (int u = 0; u < MAPS; ++u) {
    const T* keys = cache + (size_t)(kvh * MAPS + u) * a.dk;
    float* acc = acc0 + u * a.dv;
    for (int d = tid; d < a.dk; d += 256) qs[d] = load_f32(q + ((size_t)blockIdx.x * MAPS + u) * a.dk + d);
    for (int d = tid; d < a.dv; d += 256) acc[d] = 0.f;
    float m = NEG_SENTINEL, l = 0.f;
    if (KIND != SIGMOID && a.sink) {
      m = a.sink[head];
      l = 1.f;
    }
    for (int j0 = lo; j0 <= pos; j0 += 256) {
      __syncthreads();
      const int key = j0 + tid;
      float s = NEG_SENTINEL;
      long row = -1;
      if (key <= pos) row = cache_row(b, seq, key);
      if (row >= 0) {
        float dot = 0.f;
        for (int d = 0; d < a.dk; ++d) dot = fmaf(qs[d], load_f32(keys + row * width + d), dot);
        s = dot * a.scale - slope * (float)(pos - key) + bias;
        if (KIND == CAPPED) s = a.cap * tanhf(s / a.cap);
      }
      at[tid] = row;
      float corr = 1.f;
      if (KIND == SIGMOID) {
        p[tid] = s <= NEG_THRESHOLD ? 0.f : 1.f / (1.f + expf(fminf(-s, 80.f)));
        __syncthreads();  // p and at are written
      } else {
        const float mx = wave_reduce_max(s);
        if ((tid & 63) == 0) red[tid >> 6] = mx;
        __syncthreads();
        const float m_new = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
        corr = m <= NEG_THRESHOLD ? 0.f : expf(m - m_new);
        const float e = s <= NEG_THRESHOLD ? 0.f : expf(s - m_new);
        p[tid] = e;
        __syncthreads();  // red is read, p and at are written
        const float sum = wave_reduce_sum(e);
        if ((tid & 63) == 0) red[tid >> 6] = sum;
        __syncthreads();
        l = l * corr + ((red[0] + red[1]) + (red[2] + red[3]));
        m = m_new;
      }
      const int n = min(256, pos - j0 + 1);
      for (int d = tid; d < a.dv; d += 256) {
        float o = acc[d] * corr;
        for (int j = 0; j < n; ++j)
          if (at[j] >= 0) o = fmaf(p[j], load_f32(vals + at[j] * width + d), o);
        acc[d] = o;
      }
    }
    const float inv_l = KIND == SIGMOID ? 1.f : l > 0.f ? 1.f / l : 0.f;
    for (int d = tid; d < a.dv; d += 256) acc[d] *= inv_l;
    __syncthreads();  // qs, p and at are read
  }
  float inv = 1.f;
  if (MAPS == 2) {
    float ss = 0.f;
    for (int d = tid; d < a.dv; d += 256) {
      const float o = acc0[d] - a.share * acc0[a.dv + d];
      acc0[d] = o;
      ss = fmaf(o, o, ss);
    }
    ss = wave_reduce_sum(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    inv = a.factor / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / a.vdim + a.eps);
  }
  for (int d = tid; d < a.dv; d += 256) write_gated(g, a, tok, head, d, acc0[d] * inv);
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

static AttnShape attn_shape(int64_t heads, int64_t kv_heads, int64_t maps, int64_t dk, int64_t dv,
                            const torch::Tensor& cache) {
  TORCH_CHECK(kv_heads >= 1 && heads >= 1 && heads % kv_heads == 0 && dk % 32 == 0 && dv % 16 == 0 && dk > 0 && dv > 0);
  TORCH_CHECK(cache.size(2) == kv_heads * (maps * dk + dv), "cache width mismatch");
  AttnShape a{};
  a.heads = heads, a.kv_heads = kv_heads, a.dk = dk, a.dv = dv;
  a.scale = 1.f;
  return a;
}

// out: a view [T, >= heads * dv] with unit column stride; gate: [T, heads * dv] or [T, heads], likewise, in out's dtype
static GatedOut gated_out(const torch::Tensor& out, const c10::optional<torch::Tensor>& gate, int64_t t,
                          const AttnShape& a) {
  const bool f32 = f32_or_bf16(out);
  TORCH_CHECK(out.dim() == 2 && out.stride(1) == 1 && out.size(0) == t && out.size(1) >= (long)a.heads * a.dv);
  const bool by4 = out.stride(0) % 4 == 0 && reinterpret_cast<uintptr_t>(out.data_ptr()) % 16 == 0;
  GatedOut g{out.data_ptr(), out.stride(0), nullptr, 0, false, f32, by4};
  if (gate.has_value()) {
    TORCH_CHECK(gate->is_cuda() && gate->dim() == 2 && gate->stride(1) == 1 && gate->dtype() == out.dtype());
    g.per_head = gate->size(1) == a.heads;
    TORCH_CHECK(gate->size(0) == t && (g.per_head || gate->size(1) == (long)a.heads * a.dv));
    g.gate = gate->data_ptr();
    g.gate_stride = gate->stride(0);
  }
  return g;
}

template <typename K>
static void allow_lds(K kernel, size_t lds) {
  if (lds <= 65536) return;
  TORCH_CHECK(lds <= 160 * 1024, "LDS request of ", lds, " bytes");
  const hipError_t e =
      hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  TORCH_CHECK(e == hipSuccess, "LDS request refused: ", hipGetErrorString(e));
}

template <int KIND, int MAPS, int RC, int VB, int QB>
static void launch_tiles(dim3 grid, const torch::Tensor& q, const torch::Tensor& cache, GatedOut g, float* po,
                         float* pml, const int* tiles, PagedRows b, AttnShape a, int n_splits) {
  constexpr int KT = MAPS * RC * 32 + VB * 16 <= 512 ? 64 : 32;
  static_assert(PAGE % KT == 0, "a tile lies in one page");
  const size_t lds = 2 * KT * (MAPS * RC * 32 + VB * 16 + 2 * TPAD) * 2;
  allow_lds(&paged_attn_kernel<KIND, MAPS, RC, VB, QB, KT>, lds);
  paged_attn_kernel<KIND, MAPS, RC, VB, QB, KT><<<grid, 256, lds, c10::hip::getCurrentHIPStream().stream()>>>(
      BF16P(q), BF16P(cache), g, po, pml, tiles, b, a, (int)q.size(0), n_splits);
}

// blocks of 16 rows that a wave takes of `rows` rows of a token run: two share the reading of a tile
template <int MAPS>
static int row_blocks(int rows, int dk, int dv) {
  return MAPS == 1 && rows >= 128 && dk <= 128 && dv <= 128 ? 2 : 1;
}

template <int KIND, int MAPS, int RC, int VB>
static void launch_attn(bool decode, int blocks, dim3 grid, const torch::Tensor& q, const torch::Tensor& cache,
                        GatedOut g, float* po, float* pml, const int* tiles, PagedRows b, AttnShape a, int n_splits) {
  if (decode) {
    const size_t tile = 4 * KVT * (VB * 16 + TPAD) * 2;
    const size_t merge = MAPS * (4 * 16 * 2 + 4 * (size_t)(a.heads / a.kv_heads) * a.dv) * 4;
    const size_t lds = std::max(tile, merge);
    allow_lds(&paged_attn_decode<KIND, MAPS, RC, VB>, lds);
    paged_attn_decode<KIND, MAPS, RC, VB><<<grid, 256, lds, c10::hip::getCurrentHIPStream().stream()>>>(
        BF16P(q), BF16P(cache), g, po, pml, b, a, (int)q.size(0), n_splits);
    return;
  }
  if constexpr (MAPS == 1 && RC <= 4 && VB <= 8) {
    if (blocks == 2) return launch_tiles<KIND, MAPS, RC, VB, 2>(grid, q, cache, g, po, pml, tiles, b, a, n_splits);
  }
  launch_tiles<KIND, MAPS, RC, VB, 1>(grid, q, cache, g, po, pml, tiles, b, a, n_splits);
}

// q [T, H, dk] or [T, H, 2, dk] in the cache's dtype; tiles [n, 2] int32 runs of at most
// run_tokens tokens; max_keys: most keys that any row sees. `a` and `g` are complete.
template <int KIND, int MAPS>
static void run_attention(const torch::Tensor& q, const torch::Tensor& cache, const torch::Tensor& pos,
                          const torch::Tensor& owner, const torch::Tensor& tables, const torch::Tensor& tiles,
                          int64_t run_tokens, int64_t max_keys, const AttnShape& a, const GatedOut& g, int64_t splits) {
  const bool f32 = f32_or_bf16(q);
  const long t = q.size(0);
  TORCH_CHECK(q.is_contiguous() && q.dtype() == cache.dtype() && q.numel() == t * a.heads * MAPS * a.dk);
  const PagedRows b = paged_rows(pos, owner, tables, cache, t);
  if (t == 0) return;
  auto stream = c10::hip::getCurrentHIPStream().stream();
  if (f32 || a.dk > 256 || a.dv > 256) {
    const size_t lds = ((size_t)a.dk + MAPS * a.dv + 256) * 4 + 256 * 8;
    TORCH_CHECK(lds <= 65536, "head sizes ", a.dk, " and ", a.dv, " are not supported");
    if (f32) {
      paged_attn_simple<KIND, MAPS, float>
          <<<t * a.heads, 256, lds, stream>>>(q.data_ptr<float>(), cache.data_ptr<float>(), g, b, a);
    } else {
      paged_attn_simple<KIND, MAPS, unsigned short><<<t * a.heads, 256, lds, stream>>>(BF16P(q), BF16P(cache), g, b, a);
    }
    HIP_CHECK_LAST();
    return;
  }
  TORCH_CHECK(splits <= 64 && run_tokens >= 1, "at most 64 key splits");
  TORCH_CHECK(tiles.is_cuda() && tiles.dtype() == torch::kInt32 && tiles.is_contiguous() && tiles.dim() == 2);
  const int group = a.heads / a.kv_heads;
  const bool decode = run_tokens == 1 && group <= 16 && tiles.size(0) == t;
  const int blocks = decode ? 1 : row_blocks<MAPS>((int)run_tokens * group, a.dk, a.dv);
  const int row_groups = ((int)run_tokens * group + 64 * blocks - 1) / (64 * blocks);
  dim3 grid(tiles.size(0), a.kv_heads * (decode ? 1 : row_groups), 1);
  int n_splits = (int)splits;
  if (n_splits <= 0) {
    // enough workgroups for the chip; a decoding workgroup reads 4 tiles at once
    const long tiles_per = decode ? 4 : 1, wanted = decode ? 512 : 256;
    const long wgs = (long)grid.x * grid.y;
    n_splits = (int)std::max(
        1L, std::min({(long)((max_keys + KVT * tiles_per - 1) / (KVT * tiles_per)), wanted / std::max(1L, wgs), 64L}));
  }
  grid.z = n_splits;
  const bool parts = n_splits > 1 || (decode && MAPS > 1);
  auto f32o = q.options().dtype(torch::kFloat32);
  auto part_o = torch::empty({parts ? (long)n_splits * t * a.heads * MAPS * a.dv : 0}, f32o);
  auto part_ml = torch::empty({parts ? (long)n_splits * t * a.heads * MAPS * 2 : 0}, f32o);
  float* po = parts ? part_o.data_ptr<float>() : nullptr;
  float* pml = parts ? part_ml.data_ptr<float>() : nullptr;
#define PA(RC, VB) \
  launch_attn<KIND, MAPS, RC, VB>(decode, blocks, grid, q, cache, g, po, pml, tiles.data_ptr<int>(), b, a, n_splits)
#define PAV(RC)              \
  do {                       \
    if (a.dv <= 32) PA(RC, 2); \
    else if (a.dv <= 64) PA(RC, 4); \
    else if (a.dv <= 128) PA(RC, 8); \
    else PA(RC, 16);         \
  } while (0)
  if (a.dk <= 32) PAV(1);
  else if (a.dk <= 64) PAV(2);
  else if (a.dk <= 128) PAV(4);
  else PAV(8);
#undef PAV
#undef PA
  HIP_CHECK_LAST();
  if (parts) {
    paged_attn_combine<KIND, MAPS><<<t * a.heads, COMBINE_THREADS(MAPS), 0, stream>>>(po, pml, g, a, t * a.heads, n_splits);
    HIP_CHECK_LAST();
  }
}
