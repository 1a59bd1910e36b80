// Latent (MLA-style) attention over a paged cache for CDNA4 (gfx950).
//
// The cache holds one latent row c (RP values) per token and nothing per head.
// Queries arrive already carried into latent space (q' = W_uk^T q), so a score
// is q'.c and the weighted sum of c is carried to value space afterwards: all
// heads of a token attend over ONE shared key/value row, i.e. multi-query
// attention with head size RP. (token, head) pairs of a run of tokens are the
// rows of an mfma_f32_16x16x32_bf16 tile, so a staged latent tile serves every
// head and every token of the run.
//
// A cached row may be longer than what is summed: its first VP values are keys
// and values, the rest (a rotated part that all heads share) are keys only.
//
//   latent_attn_kernel     MFMA flash kernel, prompts and decoding, ragged
//                          batches, sliding window, optional key split; a sink in
//                          the softmax and a factor per head on the result
//   latent_attn_combine    merges key splits
//   latent_attn_simple     any latent size, 32-bit or bf16 storage
//   latent_write           RMS-normalises new latents into their pages
//
// Rows, positions and page tables come from device memory; every page index is
// checked against the pool before it is used.

#include "common.h"
#include "paged.h"
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>

#define LKVT 32   // keys per staged tile; tiles are aligned, so one lies in one page
#define LOG2E 1.4426950408889634f

// LDS row padding (elements): 16, or 8 where two workgroups would not fit in a CU otherwise
constexpr int lds_pad(int rc) { return rc > 16 ? 8 : 16; }

// what is done to a row's weighted sum at the end
struct LatentEnd {
  const float* sink;    // [H] score of one more entry of the softmax, without a value; or null
  const float* factor;  // [T, H] or null
};

// factor of sum_j exp2(s_j - m) v_j, given l = sum_j exp2(s_j - m)
__device__ __forceinline__ float end_factor(const LatentEnd& e, size_t flat, int heads, float m, float l) {
  float f = l > 0.f ? 1.f / l : 0.f;
  if (e.sink) {
    const float s = e.sink[flat % heads] * LOG2E, mx = fmaxf(m, s), w = exp2f(m - mx);
    f = w / fmaf(l, w, exp2f(s - mx));
  }
  return e.factor ? f * e.factor[flat] : f;
}

// ------------------------------------------------------------ MFMA kernel

// A workgroup is 4 waves = RG groups of 16 rows x DG slices of the latent's
// dims: DG > 1 when there are few rows (decoding), so that all waves share the
// staging and the weighted sum. Tiles are double-buffered in LDS and the next
// one is loaded while the current one is used. The same staged tile is the keys
// (row-major fragments) and the values (transposing LDS loads).
//
// RC = row size in 32-wide MFMA k-chunks (columns past RP read as zero), VC = those
// of them that are values. Grid: (token runs, groups of 16*RG rows, key splits).
template <int RC, int VC, int DG>
__global__ __launch_bounds__(256) void latent_attn_kernel(
    const unsigned short* __restrict__ q,      // [T, H, RP]
    const unsigned short* __restrict__ cache,  // [num_pages, PAGE, RP]
    unsigned short* __restrict__ out,          // [T, H, VP] (n_splits == 1)
    float* __restrict__ part_o,                // [n_splits, T*H, VP]
    float* __restrict__ part_ml,               // [n_splits, T*H, 2]
    const int* __restrict__ tiles,             // [n, 2] first token, token count
    PagedRows b,
    int total_tokens,
    int heads,
    int rp,
    int vp,
    int window,
    float scale_log2e,
    int n_splits,
    LatentEnd end) {
  constexpr int R = RC * 32;
  constexpr int RG = 4 / DG;
  constexpr int ROW = R + lds_pad(RC);           // LDS row in elements
  constexpr int LOADS = LKVT * (R / 8);          // 16-byte loads per tile
  constexpr int NLD = (LOADS + 255) / 256;       // per thread
  constexpr int DB = (VC * 2 + DG - 1) / DG;     // 16-wide dim blocks per wave
  const int tok0 = tiles[2 * blockIdx.x];
  const int ntok = tiles[2 * blockIdx.x + 1];
  const int rows = ntok * heads;
  const int g0 = blockIdx.y * 16 * RG;  // first row of this workgroup
  if (g0 >= rows) return;               // uniform over the workgroup
  const int g1 = min(g0 + 16 * RG, rows);

  const int tid = threadIdx.x;
  const int wave = tid / WAVE;
  const int lane = tid & (WAVE - 1);
  const int col = lane & 15;
  const int hi = lane >> 4;
  const int r0 = g0 + (wave / DG) * 16;  // first row of this wave
  const int d0 = (wave % DG) * DB;       // first dim block of this wave

  extern __shared__ unsigned short smem[];
  unsigned short* p_lds = smem + 2 * LKVT * ROW + wave * 16 * (LKVT + 8);

  const int seq = b.owner[tok0];
  const int first_pos = b.pos[tok0 + g0 / heads];
  const int last_pos = b.pos[tok0 + (g1 - 1) / heads];
  const int key_lo = window > 0 ? max(0, first_pos - window + 1) / LKVT * LKVT : 0;
  const int key_hi = last_pos + 1;
  const int n_tiles = (key_hi - key_lo + LKVT - 1) / LKVT;
  const int per_split = (n_tiles + n_splits - 1) / n_splits;
  const int j_begin = key_lo + blockIdx.z * per_split * LKVT;
  const int j_end = min(key_hi, j_begin + per_split * LKVT);

  bf16x8 q_frag[RC];
  {
    const int row = r0 + col;
    const unsigned short* src = q + ((size_t)tok0 * heads + row) * rp;
#pragma unroll
    for (int kc = 0; kc < RC; ++kc) {
      const int c0 = kc * 32 + hi * 8;
      if (row < rows && c0 < rp)
        q_frag[kc] = *reinterpret_cast<const bf16x8*>(src + c0);
      else
        q_frag[kc] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
    }
  }

  f32x4 acc_o[DB];
  float m_row[4], l_row[4];  // l_row: this lane's share of the row's sum
  int row_pos[4], row_lo[4];
#pragma unroll
  for (int d = 0; d < DB; ++d) acc_o[d] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    m_row[r] = NEG_SENTINEL;
    l_row[r] = 0.f;
    const int row = r0 + hi * 4 + r;
    row_pos[r] = row < rows ? b.pos[tok0 + row / heads] : -1;  // -1: sees nothing
    row_lo[r] = window > 0 ? row_pos[r] - window + 1 : 0;
  }
  // keys that every row of this wave sees: [all_lo, all_hi]
  const bool full_wave = r0 + 16 <= rows;
  const int all_hi = full_wave ? b.pos[tok0 + r0 / heads] : -1;
  const int all_lo = full_wave && window > 0 ? b.pos[tok0 + (r0 + 15) / heads] - window + 1 : 0;

  bf16x8 next[NLD];
  // rows of tile j0 that lie in [0, j_end); zero elsewhere and past rp
  auto fetch = [&](int j0) {
    const long at = cache_row(b, seq, j0);
#pragma unroll
    for (int i = 0; i < NLD; ++i) {
      const int idx = tid + i * 256;
      const int row = idx / (R / 8);
      const int c8 = (idx - row * (R / 8)) * 8;
      next[i] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
      if ((LOADS % 256 == 0 || idx < LOADS) && at >= 0 && j0 + row < j_end && c8 < rp)
        next[i] = *reinterpret_cast<const bf16x8*>(cache + ((size_t)at + row) * rp + c8);
    }
  };
  auto stage = [&](unsigned short* buf) {
#pragma unroll
    for (int i = 0; i < NLD; ++i) {
      const int idx = tid + i * 256;
      const int row = idx / (R / 8);
      const int c8 = (idx - row * (R / 8)) * 8;
      if (LOADS % 256 == 0 || idx < LOADS) *reinterpret_cast<bf16x8*>(&buf[row * ROW + c8]) = next[i];
    }
  };

  if (j_begin < j_end) {
    fetch(j_begin);
    stage(smem);
  }
  __syncthreads();
  int which = 0;
  for (int j0 = j_begin; j0 < j_end; j0 += LKVT, which ^= 1) {
    const unsigned short* k_lds = smem + which * LKVT * ROW;
    const bool more = j0 + LKVT < j_end;
    if (more) fetch(j0 + LKVT);

    f32x4 s_acc[2];
#pragma unroll
    for (int nb = 0; nb < 2; ++nb) {
      s_acc[nb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kc = 0; kc < RC; ++kc) {
        const bf16x8 kt = *reinterpret_cast<const bf16x8*>(&k_lds[(nb * 16 + col) * ROW + kc * 32 + hi * 8]);
        s_acc[nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(q_frag[kc], kt, s_acc[nb], 0, 0, 0);
      }
    }

    const bool interior = j0 >= all_lo && j0 + LKVT - 1 <= all_hi && j0 + LKVT <= j_end;
    float corr[4], p[2][4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      // masking and the running max stay in separate loops (see prefill_attn.hip)
      float s[2];
#pragma unroll
      for (int nb = 0; nb < 2; ++nb) s[nb] = s_acc[nb][r] * scale_log2e;
      if (!interior) {
#pragma unroll
        for (int nb = 0; nb < 2; ++nb) {
          const int key = j0 + nb * 16 + col;
          if (key >= j_end || key > row_pos[r] || key < row_lo[r]) s[nb] = NEG_SENTINEL;
        }
      }
      float mx = fmaxf(s[0], s[1]);
#pragma unroll
      for (int off = 8; off > 0; off >>= 1) mx = fmaxf(mx, __shfl_xor(mx, off, WAVE));
      const float m_new = fmaxf(m_row[r], mx);
      corr[r] = (m_row[r] <= NEG_THRESHOLD) ? 0.f : exp2f(m_row[r] - m_new);
#pragma unroll
      for (int nb = 0; nb < 2; ++nb) p[nb][r] = (s[nb] <= NEG_THRESHOLD) ? 0.f : exp2f(s[nb] - m_new);
      l_row[r] = l_row[r] * corr[r] + (p[0][r] + p[1][r]);
      m_row[r] = m_new;
    }
    // P to A-fragment layout through this wave's own LDS
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int nb = 0; nb < 2; ++nb) p_lds[(hi * 4 + r) * (LKVT + 8) + nb * 16 + col] = f32_to_bf16(p[nb][r]);
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    const bf16x8 p_frag = *reinterpret_cast<const bf16x8*>(&p_lds[col * (LKVT + 8) + hi * 8]);

    const unsigned short* v_lds = k_lds + (hi * 8 + col / 4) * ROW + (col & 3) * 4;
#pragma unroll
    for (int d = 0; d < DB; ++d) {
      if (VC * 2 % DG != 0 && d0 + d >= VC * 2) break;  // uniform over the wave
#pragma unroll
      for (int r = 0; r < 4; ++r) acc_o[d][r] *= corr[r];
      acc_o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
          p_frag, load_keys(v_lds + (d0 + d) * 16, ROW), acc_o[d], 0, 0, 0);
    }
    if (more) stage(smem + (which ^ 1) * LKVT * ROW);
    __syncthreads();
  }

#pragma unroll
  for (int r = 0; r < 4; ++r) {
    float l = l_row[r];
#pragma unroll
    for (int off = 8; off > 0; off >>= 1) l += __shfl_xor(l, off, WAVE);
    const int row = r0 + hi * 4 + r;
    if (row >= rows) continue;
    const size_t flat = (size_t)tok0 * heads + row;
    if (n_splits == 1) {
      const float f = end_factor(end, flat, heads, m_row[r], l);
#pragma unroll
      for (int d = 0; d < DB; ++d) {
        const int c = (d0 + d) * 16 + col;
        if (c < vp) out[flat * vp + c] = f32_to_bf16(acc_o[d][r] * f);
      }
    } else {
      const size_t at = (size_t)blockIdx.z * total_tokens * heads + flat;
#pragma unroll
      for (int d = 0; d < DB; ++d) {
        const int c = (d0 + d) * 16 + col;
        if (c < vp) part_o[at * vp + c] = acc_o[d][r];
      }
      if (col == 0 && wave % DG == 0) {
        part_ml[at * 2] = m_row[r];
        part_ml[at * 2 + 1] = l;
      }
    }
  }
}

// one workgroup per (token, head) row and 128 of its dims
__global__ __launch_bounds__(128) void latent_attn_combine(
    const float* __restrict__ part_o, const float* __restrict__ part_ml,
    unsigned short* __restrict__ out, int n_rows, int heads, int vp, int n_splits,
    LatentEnd end) {
  __shared__ float share[WAVE];  // weight of each split in the row
  const int row = blockIdx.x;
  if (threadIdx.x < WAVE) {
    const int s = threadIdx.x;
    float m = NEG_SENTINEL, l = 0.f;
    if (s < n_splits) {
      m = part_ml[((size_t)s * n_rows + row) * 2];
      l = part_ml[((size_t)s * n_rows + row) * 2 + 1];
    }
    const float mx = wave_reduce_max(m);
    const float w = m > NEG_THRESHOLD ? exp2f(m - mx) : 0.f;
    share[s] = w * end_factor(end, row, heads, mx, wave_reduce_sum(w * l));
  }
  __syncthreads();
  const int d = blockIdx.y * blockDim.x + threadIdx.x;
  if (d < vp) {
    const float* src = part_o + (size_t)row * vp + d;
    const size_t step = (size_t)n_rows * vp;
    float o[4] = {0.f, 0.f, 0.f, 0.f};
    int s = 0;
    for (; s + 4 <= n_splits; s += 4)
#pragma unroll
      for (int u = 0; u < 4; ++u) o[u] = fmaf(src[(s + u) * step], share[s + u], o[u]);
    for (; s < n_splits; ++s) o[0] = fmaf(src[s * step], share[s], o[0]);
    out[(size_t)row * vp + d] = f32_to_bf16((o[0] + o[1]) + (o[2] + o[3]));
  }
}

// ---------------------------------------------------------- simple kernel

// one workgroup of 256 per (token, head): a key per thread for the scores, a
// latent dimension per thread for the sum
template <typename T>
__global__ __launch_bounds__(256) void latent_attn_simple(
    const T* __restrict__ q,      // [T, H, RP]
    const T* __restrict__ cache,  // [num_pages, PAGE, RP]
    T* __restrict__ out,          // [T, H, VP]
    PagedRows b, int heads, int rp, int vp, int window, float scale, LatentEnd end) {
  extern __shared__ float sm[];
  float* qs = sm;           // [rp]
  float* acc = qs + rp;     // [vp, rounded up to even]
  float* p = acc + (vp + 1) / 2 * 2;  // [256]
  long* at = reinterpret_cast<long*>(p + 256);  // [256]
  __shared__ float red[4];
  const int tid = threadIdx.x;
  const int tok = blockIdx.x / heads;
  const int seq = b.owner[tok];
  const int pos = b.pos[tok];
  const int lo = window > 0 ? max(0, pos - window + 1) : 0;
  for (int d = tid; d < rp; d += 256) qs[d] = load_f32(q + (size_t)blockIdx.x * rp + d);
  for (int d = tid; d < vp; d += 256) acc[d] = 0.f;
  float m = NEG_SENTINEL, l = 0.f;
  for (int j0 = lo; j0 <= pos; j0 += 256) {
    __syncthreads();
    const int key = j0 + tid;
    float s = NEG_SENTINEL;
    long row = -1;
    if (key <= pos) row = cache_row(b, seq, key);
    if (row >= 0) {
      float dot = 0.f;
      for (int d = 0; d < rp; ++d) dot = fmaf(qs[d], load_f32(cache + (size_t)row * rp + d), dot);
      s = dot * scale;
    }
    at[tid] = row;
    float mx = wave_reduce_max(s);
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
    for (int d = tid; d < vp; d += 256) {
      float o = acc[d] * corr;
      for (int j = 0; j < n; ++j)
        if (at[j] >= 0) o = fmaf(p[j], load_f32(cache + (size_t)at[j] * rp + d), o);
      acc[d] = o;
    }
  }
  const float f = end_factor(end, blockIdx.x, heads, m * LOG2E, l);
  for (int d = tid; d < vp; d += 256) store_f32(out + (size_t)blockIdx.x * vp + d, acc[d] * f);
}

// ---------------------------------------------------------- latent writing

// c = y / sqrt(mean(y^2) + eps) * w of one token, stored at its place
template <typename TY, typename TC>
__global__ __launch_bounds__(256) void latent_write_kernel(
    const TY* __restrict__ y, int y_stride,  // [T, y_stride], rank values each
    const float* __restrict__ w,             // [rank]
    TC* __restrict__ cache, PagedRows b, int rank, int rp, float eps) {
  __shared__ float red[4];
  const int tid = threadIdx.x;
  const TY* row = y + (size_t)blockIdx.x * y_stride;
  float ss = 0.f;
  for (int d = tid; d < rank; d += 256) {
    const float v = load_f32(row + d);
    ss = fmaf(v, v, ss);
  }
  ss = wave_reduce_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  const float inv = 1.f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / rank + eps);
  const long at = cache_row(b, b.owner[blockIdx.x], b.pos[blockIdx.x]);
  if (at < 0) return;
  for (int d = tid; d < rp; d += 256)
    store_f32(cache + (size_t)at * rp + d, d < rank ? load_f32(row + d) * inv * w[d] : 0.f);
}

// ------------------------------------------------------------------- host

template <int RC, int VC, int DG>
static void launch_mfma(dim3 grid, const torch::Tensor& q, const torch::Tensor& cache, torch::Tensor& out,
                        torch::Tensor& part_o, torch::Tensor& part_ml, const torch::Tensor& tiles, PagedRows b,
                        int heads, int rp, int vp, int window, float scale, int n_splits, LatentEnd end) {
  constexpr size_t lds = (2 * LKVT * (RC * 32 + lds_pad(RC)) + 4 * 16 * (LKVT + 8)) * 2;
  static bool allowed = false;
  if (lds > 65536 && !allowed) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_attn_kernel<RC, VC, DG>),
                                       hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    TORCH_CHECK(e == hipSuccess, "LDS request refused: ", hipGetErrorString(e));
    allowed = true;
  }
  latent_attn_kernel<RC, VC, DG><<<grid, 256, lds, at::cuda::getCurrentCUDAStream()>>>(
      BF16P(q), BF16P(cache), BF16P(out), part_o.numel() ? part_o.data_ptr<float>() : nullptr,
      part_ml.numel() ? part_ml.data_ptr<float>() : nullptr, tiles.data_ptr<int>(), b, (int)q.size(0), heads, rp, vp,
      window, scale * LOG2E, n_splits, end);
}

torch::Tensor latent_attention(
    torch::Tensor q,       // [T, H, RP] bf16 or f32
    torch::Tensor cache,   // [pages, PAGE, RP], dtype of q
    torch::Tensor pos, torch::Tensor owner, torch::Tensor tables,
    torch::Tensor tiles,   // [n, 2] int32 runs of at most run_tokens tokens
    int64_t run_tokens,
    int64_t max_keys,      // most keys that any row sees
    int64_t window, double scale, int64_t splits,
    int64_t values,        // size of the result: the first values of a row, 0 for all of them
    c10::optional<torch::Tensor> sink,      // [H] f32
    c10::optional<torch::Tensor> factor) {  // [T, H] f32
  TORCH_CHECK(q.is_cuda() && q.dim() == 3 && q.is_contiguous() && q.dtype() == cache.dtype());
  const int t = q.size(0), heads = q.size(1), rp = q.size(2), vp = values > 0 ? (int)values : rp;
  TORCH_CHECK(cache.size(2) == rp && rp % 32 == 0 && vp <= rp, "latent width mismatch");
  const PagedRows b = paged_rows(pos, owner, tables, cache, t);
  LatentEnd end{nullptr, nullptr};
  auto f32_values = [](const c10::optional<torch::Tensor>& x, long n) -> const float* {
    if (!x.has_value()) return nullptr;
    TORCH_CHECK(x->is_cuda() && x->dtype() == torch::kFloat32 && x->is_contiguous() && x->numel() == n);
    return x->data_ptr<float>();
  };
  end.sink = f32_values(sink, heads);
  end.factor = f32_values(factor, (long)t * heads);
  auto out = torch::empty({t, heads, vp}, q.options());
  if (t == 0) return out;
  auto stream = at::cuda::getCurrentCUDAStream();
  const bool f32 = q.dtype() == torch::kFloat32;
  TORCH_CHECK(f32 || q.dtype() == torch::kBFloat16);
  if (f32 || rp > 18 * 32 || vp > 16 * 32) {
    const size_t lds = ((size_t)rp + (vp + 1) / 2 * 2 + 256) * 4 + 256 * 8;
    TORCH_CHECK(lds <= 65536, "latent size ", rp, " is not supported");
    if (f32)
      latent_attn_simple<float><<<t * heads, 256, lds, stream>>>(
          q.data_ptr<float>(), cache.data_ptr<float>(), out.data_ptr<float>(), b, heads, rp, vp, (int)window,
          (float)scale, end);
    else
      latent_attn_simple<unsigned short><<<t * heads, 256, lds, stream>>>(
          BF16P(q), BF16P(cache), BF16P(out), b, heads, rp, vp, (int)window, (float)scale, end);
    HIP_CHECK_LAST();
    return out;
  }
  TORCH_CHECK(splits <= 64, "at most 64 key splits");
  TORCH_CHECK(tiles.is_cuda() && tiles.dtype() == torch::kInt32 && tiles.is_contiguous() && tiles.dim() == 2);
  const int rows = (int)run_tokens * heads;
  const int rg = rows <= 16 ? 1 : rows <= 32 ? 2 : 4;  // 16-row groups per workgroup
  dim3 grid(tiles.size(0), (rows + 16 * rg - 1) / (16 * rg), 1);
  int n_splits = (int)splits;
  if (n_splits <= 0) {
    // enough workgroups for the chip
    const long wgs = (long)grid.x * grid.y;
    n_splits = (int)std::max(1L, std::min({(long)((max_keys + LKVT - 1) / LKVT), 128 / std::max(1L, wgs), 64L}));
  }
  grid.z = n_splits;
  auto f32o = q.options().dtype(torch::kFloat32);
  auto part_o = torch::empty({n_splits > 1 ? (long)n_splits * t * heads * vp : 0}, f32o);
  auto part_ml = torch::empty({n_splits > 1 ? (long)n_splits * t * heads * 2 : 0}, f32o);
#define LA2(RC, VC, DG)                                                                                              \
  launch_mfma<RC, VC, DG>(grid, q, cache, out, part_o, part_ml, tiles, b, heads, rp, vp, (int)window, (float)scale, \
                          n_splits, end)
#define LA(RC, VC)                    \
  do {                                \
    if (rg == 1) LA2(RC, VC, 4);      \
    else if (rg == 2) LA2(RC, VC, 2); \
    else LA2(RC, VC, 1);              \
  } while (0)
  const int rc = rp / 32, vc = (vp + 31) / 32;
  if (rc <= 1) LA(1, 1);
  else if (rc <= 2 && vc <= 1) LA(2, 1);
  else if (rc <= 2) LA(2, 2);
  else if (rc <= 3 && vc <= 2) LA(3, 2);
  else if (rc <= 3) LA(3, 3);
  else if (rc <= 4) LA(4, 4);
  else if (rc <= 5 && vc <= 4) LA(5, 4);
  else if (rc <= 6) LA(6, 6);
  else if (rc <= 8) LA(8, 8);
  else if (rc <= 10 && vc <= 8) LA(10, 8);
  else if (rc <= 12) LA(12, 12);
  else if (rc <= 14 && vc <= 12) LA(14, 12);
  else if (rc <= 16) LA(16, 16);
  else LA(18, 16);
#undef LA
#undef LA2
  HIP_CHECK_LAST();
  if (n_splits > 1) {
    latent_attn_combine<<<dim3(t * heads, (vp + 127) / 128), 128, 0, stream>>>(
        part_o.data_ptr<float>(), part_ml.data_ptr<float>(), BF16P(out), t * heads, heads, vp, n_splits, end);
    HIP_CHECK_LAST();
  }
  return out;
}

void latent_write(
    torch::Tensor y,      // [T, >= offset + rank] f32 or bf16; columns [offset, offset + rank)
    int64_t offset,
    torch::Tensor w,      // [rank] f32
    torch::Tensor cache, torch::Tensor pos, torch::Tensor owner, torch::Tensor tables, double eps) {
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous());
  TORCH_CHECK(w.is_cuda() && w.dtype() == torch::kFloat32 && w.is_contiguous());
  const int rank = w.numel(), rp = cache.size(2), stride = y.size(1), t = y.size(0);
  TORCH_CHECK(rank <= rp && offset + rank <= stride, "latent sizes do not fit");
  const PagedRows b = paged_rows(pos, owner, tables, cache, t);
  auto stream = at::cuda::getCurrentCUDAStream();
  const bool yf = y.dtype() == torch::kFloat32, cf = cache.dtype() == torch::kFloat32;
  TORCH_CHECK((yf || y.dtype() == torch::kBFloat16) && (cf || cache.dtype() == torch::kBFloat16));
#define LW(TY, TC, YP, CP) \
  latent_write_kernel<TY, TC><<<t, 256, 0, stream>>>(YP + offset, stride, w.data_ptr<float>(), CP, b, rank, rp, (float)eps)
  if (yf && cf) LW(float, float, y.data_ptr<float>(), cache.data_ptr<float>());
  else if (yf) LW(float, unsigned short, y.data_ptr<float>(), BF16P(cache));
  else if (cf) LW(unsigned short, float, BF16P(y), cache.data_ptr<float>());
  else LW(unsigned short, unsigned short, BF16P(y), BF16P(cache));
#undef LW
  HIP_CHECK_LAST();
}
