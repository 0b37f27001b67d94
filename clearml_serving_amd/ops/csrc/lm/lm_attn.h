// What the attention kernels of csrc/lm share: rotary positions, caps on
// scores, visible keys, and the sums of waves and key ranges meeting.
#pragma once

#include "lm_common.h"

constexpr float LM_LOG2E = 1.4426950408889634f;

// Pair p of a rotated part is (2p, 2p+1) or, with `half`, (p, p + pairs):
// (u, v) -> gain * (u cos - v sin, v cos + u sin). Elements behind the pairs
// pass unchanged.
struct Rot {
  const float* inv_freq;
  int pairs, half;
  float gain;
};

__device__ __forceinline__ void rot_places(const Rot& r, int p, int* u,
                                           int* v) {
  const bool h = r.half && p < r.pairs;
  *u = h ? p : 2 * p;
  *v = h ? p + r.pairs : 2 * p + 1;
}

// Scores in the base-2 exponent's scale: s * scale, or with a cap
// cap * tanh(s * scale / cap).
struct Score {
  float scale2;    // scale * log2 e
  float in, out2;  // scale / cap, cap * log2 e
  bool capped;
};

inline Score make_score(double scale, double cap) {
  Score s{};
  s.scale2 = (float)(scale * 1.4426950408889634);
  s.capped = cap > 0.0;
  if (s.capped) {
    s.in = (float)(scale / cap);
    s.out2 = (float)(cap * 1.4426950408889634);
  }
  return s;
}

template <typename T> __device__ __forceinline__ float cap_tanh(float z);
template <> __device__ __forceinline__ float cap_tanh<float>(float z) {
  return tanhf(z);
}
// 1 - 2 / (1 + e^2z): absolute error of a few float ulp of one, below what
// 16-bit queries and keys leave of a score
template <> __device__ __forceinline__ float cap_tanh<bf16>(float z) {
  return 1.f - 2.f * __builtin_amdgcn_rcpf(1.f + exp_f(2.f * z));
}

// A query at position `pos` sees the keys up to it, with a window the last
// `window` of them and the first `keep` of the sequence. Visible key n lies
// at position n, from number `kf` on at n + skip. With `pool` the first kf keys
// are the means of the whole blocks of so many tokens in front of the window.
struct Visible {
  int kf, skip, n;
  __device__ __forceinline__ int position(int i) const {
    return i < kf ? i : i + skip;
  }
};

__device__ __forceinline__ Visible visible_keys(int pos, int window, int keep,
                                                int pool) {
  const int lo = window > 0 ? max(0, pos - window + 1) : 0;
  Visible v;
  v.kf = pool > 0 ? lo / pool : min(keep, lo);
  v.skip = lo - v.kf;
  v.n = pos + 1 - v.skip;
  return v;
}

// The waves' sums of one query row block meet: acc[i] is C[c = 16 i + 4 g +
// r][head lane & 15], m_run the maximum (base 2) of the wave's keys, l_run the
// lane group's part of the sum of weights. `tiles`: float storage of the waves
// (wave w at tiles + w * wstep floats, 16 * (cols + 4) each), free by now.
// put(head row, column, sums, max, sum of weights) takes four columns.
template <int NT, typename Put>
__device__ __forceinline__ void meet_waves(const lm_f32x4 (&acc)[NT],
                                           float m_run, float l_run, int cols,
                                           int heads, float (*stat)[16][2],
                                           float* tiles, int wstep, Put put) {
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int r16 = lane & 15, g = lane >> 4, nw = blockDim.x >> 6;
  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  if (g == 0) {
    stat[wave][r16][0] = m_run;
    stat[wave][r16][1] = l_run;
  }
  __syncthreads();
  float m_f = -INFINITY;
  for (int w = 0; w < nw; ++w) m_f = fmaxf(m_f, stat[w][r16][0]);
  const float f = m_run == -INFINITY ? 0.f
                                     : __builtin_amdgcn_exp2f(m_run - m_f);
  const int OP = cols + 4;
  float* ow = tiles + wave * wstep;
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    if (i * 16 < cols) {
      const float v[4] = {acc[i][0] * f, acc[i][1] * f, acc[i][2] * f,
                          acc[i][3] * f};
      store4(ow + r16 * OP + i * 16 + 4 * g, v);
    }
  }
  __syncthreads();
  const int c4 = cols / 4;
  for (int i = tid; i < heads * c4; i += blockDim.x) {
    const int r = i / c4, c = (i % c4) * 4;
    float m = -INFINITY, l = 0.f;
    for (int w = 0; w < nw; ++w) m = fmaxf(m, stat[w][r][0]);
    for (int w = 0; w < nw; ++w)
      if (stat[w][r][0] != -INFINITY)
        l += stat[w][r][1] * __builtin_amdgcn_exp2f(stat[w][r][0] - m);
    lm_f32x4 o = {0.f, 0.f, 0.f, 0.f};
    for (int w = 0; w < nw; ++w)
      o += *reinterpret_cast<const lm_f32x4*>(tiles + w * wstep + r * OP + c);
    put(r, c, o, m, l);
  }
}

// 1 / (sum of weights + exp2(sink)) for sums relative to max m; without a
// sink: -inf
__device__ __forceinline__ float over_weights(float m, float l, float sink) {
  const float m_s = fmaxf(m, sink);
  const float e = __builtin_amdgcn_exp2f(m - m_s);
  return e / (l * e + __builtin_amdgcn_exp2f(sink - m_s));
}

// merge key ranges; a range without keys has m = -inf. out rows of ld_out,
// head h at h * C
template <typename T>
__global__ __launch_bounds__(128) void combine_ranges_kernel(
    const float* __restrict__ part_o, const float* __restrict__ part_ml,
    const T* __restrict__ sink, T* __restrict__ out, long ld_out, int splits,
    int H, int C, float out_scale) {
  const long th = blockIdx.x;
  const float sk = sink ? to_f32(sink[th % H]) * LM_LOG2E : -INFINITY;
  float m = sk;  // some range has a key: m ends finite
  for (int s = 0; s < splits; ++s)
    m = fmaxf(m, part_ml[(th * splits + s) * 2]);
  float l = exp2f(sk - m);
  for (int s = 0; s < splits; ++s)
    l += part_ml[(th * splits + s) * 2 + 1] *
         exp2f(part_ml[(th * splits + s) * 2] - m);
  const float inv = out_scale / l;
  for (int c = threadIdx.x * 4; c < C; c += 128 * 4) {
    float f[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s = 0; s < splits; ++s) {
      // an empty range wrote zeros and weighs exp2(-inf) = 0
      const float e = exp2f(part_ml[(th * splits + s) * 2] - m) * inv;
      const lm_f32x4 o = *reinterpret_cast<const lm_f32x4*>(
          part_o + (th * splits + s) * C + c);
#pragma unroll
      for (int r = 0; r < 4; ++r) f[r] += o[r] * e;
    }
    store4(out + (th / H) * ld_out + (th % H) * C + c, f);
  }
}

// Pages hold the rows of `tokens` tokens and behind them the means of the
// blocks of `pool` tokens that end in the page.
struct PageRows {
  int tokens, rows, pool;
  __device__ __forceinline__ int token(int page, int offset) const {
    return page * rows + offset;
  }
  __device__ __forceinline__ int pooled(int page, int offset) const {
    return page * rows + tokens + offset / pool;
  }
};

inline PageRows page_rows(long rows, long pool) {
  TORCH_CHECK(pool >= 0 && pool < (1 << 20), "lm: pooled block size");
  PageRows p{};
  p.rows = (int)rows;
  p.pool = (int)pool;
  p.tokens = (int)(pool ? rows * pool / (pool + 1) : rows);
  TORCH_CHECK(p.tokens >= 1 &&
                  p.rows == p.tokens + (pool ? (p.tokens + pool - 1) / pool
                                             : 0),
              "lm: page of ", rows, " rows");
  return p;
}

// [T, cols] view with 16-byte aligned rows
inline void lm_check_rows(const torch::Tensor& v, long T, long cols,
                          at::ScalarType type) {
  TORCH_CHECK(v.is_cuda() && v.dim() == 2 && v.size(0) == T &&
                  v.size(1) == cols && v.stride(1) == 1 &&
                  v.stride(0) % 8 == 0 && v.storage_offset() % 8 == 0 &&
                  v.scalar_type() == type,
              "lm: operand rows do not fit");
}

inline Rot make_rot(const torch::Tensor& inv_freq, double gain, bool half,
                    long room) {
  LM_CHECK_CONTIG(inv_freq);
  TORCH_CHECK(inv_freq.scalar_type() == at::kFloat);
  const long pairs = inv_freq.numel();
  TORCH_CHECK(2 * pairs <= room && pairs <= 256, "rotated size too large");
  return Rot{inv_freq.data_ptr<float>(), (int)pairs, half ? 1 : 0,
             (float)gain};
}
