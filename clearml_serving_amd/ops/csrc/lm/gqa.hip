// Grouped-query attention on paged rows: H query heads on G key/value heads.
//
// Cache row = G slices [key KD | value VD], in pages of block_size rows. A
// layer whose values are its keys before their norm caches the projection
// alone, [KD] per head, and behind the slices a float per head, the norm's
// factor of that key: the norm's weights are folded into the query and the
// score is multiplied by the factor, so a key is read once for both products.
//
// Preparation of queries and cache rows: norm per head, rotation of
// neighbouring pairs, mixing of the values with another layer's. Attention for
// few queries per sequence is here, for prompts in prompt_attn.hip. All takes
// a sliding window with kept first tokens or with the means of the blocks in
// front of it, a cap on the scores and a sink, each of them optional.
#include "lm_attn.h"

namespace {

// ------------------------------------------------------------------- //
// prepare
// ------------------------------------------------------------------- //
template <typename T>
struct GroupedPrep {
  T* q;              // [t, H * KD] in place
  const T *k, *v;    // [t, G * KD], [t, G * VD]; no v: values are keys
  long ld;           // row stride of q, k, v
  const T* first;    // [t, G * VD], null: no mixing
  long ld_first;
  float lam;
  const T *qn, *kn;  // norm weights [KD], null: no norm; of a norm over all
                     // heads [H * KD], [G * KD]
  const T *qb, *kb, *vb;  // biases, laid out as q, k and v, or null
  T* cache;
  long n_slots;
  int H, G, KD, VD, dim, row;
  float eps;
  PageRows page;
};

// cache row of a slot: page * tokens of a page + offset
template <typename T>
__device__ __forceinline__ T* cache_row(const GroupedPrep<T>& a, long slot) {
  return a.cache + (long)a.page.token((int)(slot / a.page.tokens),
                                      (int)(slot % a.page.tokens)) * a.row;
}

template <typename T>
__device__ __forceinline__ void load_biased(const T* p, const T* bias,
                                            float* f) {
  load8<T>(p, f);
  if (bias) {
    float b[8];
    load8<T>(bias, b);
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] += b[e];
  }
}

// Units of a token are its heads: H queries, G keys, G values. LPH lanes take
// a unit, 8 elements each.
template <typename T>
__global__ __launch_bounds__(256) void grouped_prep_kernel(
    GroupedPrep<T> a, const int* __restrict__ positions,
    const int* __restrict__ slots, Rot rot, int n_tok, int tokens_per_wg,
    int LPH) {
  extern __shared__ float trig[];  // [tokens][2][pairs]
  const int tid = threadIdx.x, pairs = rot.pairs;
  const int t0 = blockIdx.x * tokens_per_wg;
  for (int i = tid; i < tokens_per_wg * pairs; i += 256) {
    const int tt = i / pairs, p = i % pairs;
    if (t0 + tt >= n_tok) break;
    float s, c;
    sincosf((float)positions[t0 + tt] * rot.inv_freq[p], &s, &c);
    trig[tt * 2 * pairs + p] = rot.gain * c;
    trig[(tt * 2 + 1) * pairs + p] = rot.gain * s;
  }
  const bool same = a.v == nullptr;
  const int per_tok = 256 / tokens_per_wg;  // threads
  const int tt = tid / per_tok, lid = tid % per_tok;
  const int t = t0 + tt;
  __syncthreads();
  if (t >= n_tok) return;
  const float* cs = trig + tt * 2 * pairs;
  const float* sn = cs + pairs;
  const int c = lid % LPH * 8;
  const long slot = slots[t];
  const bool has_slot = slot >= 0 && slot < a.n_slots;
  T* crow = cache_row(a, has_slot ? slot : 0);
  const int SL = same ? a.KD : a.KD + a.VD;
  const int units = a.H + a.G + (same ? 0 : a.G);
  // the LPH lanes of a unit stay together
  for (int u = lid / LPH; u < units; u += per_tok / LPH) {
    const bool is_q = u < a.H, is_v = u >= a.H + a.G;
    const int size = is_v ? a.VD : a.KD;
    const bool mine = c < size;
    const T* src = is_q ? a.q + t * a.ld + u * a.KD
                 : is_v ? a.v + t * a.ld + (u - a.H - a.G) * a.VD
                        : a.k + t * a.ld + (u - a.H) * a.KD;
    const T* bias = is_q ? a.qb ? a.qb + u * a.KD : nullptr
                  : is_v ? a.vb ? a.vb + (u - a.H - a.G) * a.VD : nullptr
                         : a.kb ? a.kb + (u - a.H) * a.KD : nullptr;
    float f[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (mine) load_biased(src + c, bias ? bias + c : nullptr, f);
    if (is_v) {
      if (!mine || !has_slot) continue;
      const int hd = u - a.H - a.G;
      if (a.first) {
        float v1[8];
        load8<T>(a.first + t * a.ld_first + hd * a.VD + c, v1);
#pragma unroll
        for (int e = 0; e < 8; ++e)
          f[e] = (1.f - a.lam) * f[e] + a.lam * v1[e];
      }
      store8(crow + hd * SL + a.KD + c, f);
      continue;
    }
    float inv = 1.f;
    const T* w = is_q ? a.qn : a.kn;
    if (w) {
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += f[e] * f[e];
      for (int d = 1; d < LPH; d <<= 1) ss += __shfl_xor(ss, d, 64);
      inv = 1.f / sqrtf(ss / (float)a.dim + a.eps);
    }
    if (!mine) continue;
    if (!is_q && same) {
      if (!has_slot) continue;
      const int hd = u - a.H;
      store8(crow + hd * SL + c, f);
      if (c == 0) reinterpret_cast<float*>(crow + a.G * SL)[hd] = inv;
      continue;
    }
    if (w) {
      float g[8];
      load8<T>(w + c, g);
#pragma unroll
      for (int e = 0; e < 8; ++e) f[e] *= inv * g[e];
    }
    if (is_q && same && a.kn) {
      float g[8];
      load8<T>(a.kn + c, g);
#pragma unroll
      for (int e = 0; e < 8; ++e) f[e] *= g[e];
    }
    if (c < 2 * pairs) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int p = c / 2 + j;
        if (p < pairs) {
          const float x = f[2 * j], y = f[2 * j + 1];
          f[2 * j] = x * cs[p] - y * sn[p];
          f[2 * j + 1] = y * cs[p] + x * sn[p];
        }
      }
    }
    if (is_q) store8(a.q + t * a.ld + u * a.KD + c, f);
    else if (has_slot) store8(crow + (u - a.H) * SL + c, f);
  }
}

// The same where one norm runs over all heads of the queries and one over
// those of the keys: TPT threads hold a token's row [q | k | v], NV vectors
// each, until its sums are there.
template <typename T, int NV, int TPT>
__global__ __launch_bounds__(256) void grouped_prep_whole_kernel(
    GroupedPrep<T> a, const int* __restrict__ positions,
    const int* __restrict__ slots, Rot rot, int n_tok) {
  extern __shared__ float trig[];  // [tokens][2][pairs]
  __shared__ float sums[4][2];
  const int tid = threadIdx.x, pairs = rot.pairs;
  const int tt = tid / TPT, lid = tid % TPT;
  const int t = min((int)blockIdx.x * (256 / TPT) + tt, n_tok - 1);
  const bool mine = (int)blockIdx.x * (256 / TPT) + tt < n_tok;
  const int nq = a.H * a.KD, nk = a.G * a.KD, total = nq + nk + a.G * a.VD;
  const T* row = a.q + t * a.ld;
  float f[NV][8];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (lid + i * TPT) * 8;
    if (c < total) load_biased(row + c, a.qb ? a.qb + c : nullptr, f[i]);
  }
  float* cs = trig + tt * 2 * pairs;
  float* sn = cs + pairs;
  const float pos = (float)positions[t];
  for (int p = lid; p < pairs; p += TPT) {
    float sv, cv;
    sincosf(pos * rot.inv_freq[p], &sv, &cv);
    cs[p] = rot.gain * cv;
    sn[p] = rot.gain * sv;
  }
  float sq = 0.f, sk = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (lid + i * TPT) * 8;
    if (c < nq + nk) {
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += f[i][e] * f[i][e];
      if (c < nq) sq += ss;
      else sk += ss;
    }
  }
#pragma unroll
  for (int d = 1; d < 64; d <<= 1) {
    sq += __shfl_xor(sq, d, 64);
    sk += __shfl_xor(sk, d, 64);
  }
  if (TPT == 256 && (tid & 63) == 0) {
    sums[tid >> 6][0] = sq;
    sums[tid >> 6][1] = sk;
  }
  __syncthreads();
  if (TPT == 256) {
    sq = (sums[0][0] + sums[1][0]) + (sums[2][0] + sums[3][0]);
    sk = (sums[0][1] + sums[1][1]) + (sums[2][1] + sums[3][1]);
  }
  if (!mine) return;
  const float inv_q = 1.f / sqrtf(sq / ((float)a.H * a.dim) + a.eps);
  const float inv_k = 1.f / sqrtf(sk / ((float)a.G * a.dim) + a.eps);
  const long slot = slots[t];
  const bool has_slot = slot >= 0 && slot < a.n_slots;
  T* crow = cache_row(a, has_slot ? slot : 0);
  const int SL = a.KD + a.VD;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (lid + i * TPT) * 8;
    if (c >= total) continue;
    if (c >= nq + nk) {
      const int v = c - nq - nk;
      if (has_slot)
        store8(crow + v / a.VD * SL + a.KD + v % a.VD, f[i]);
      continue;
    }
    const bool is_q = c < nq;
    const int u = is_q ? c : c - nq, d = u % a.KD;
    const float inv = is_q ? inv_q : inv_k;
    float w[8];
    load8<T>((is_q ? a.qn : a.kn) + u, w);
#pragma unroll
    for (int e = 0; e < 8; ++e) f[i][e] *= inv * w[e];
    if (d < 2 * pairs) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int p = d / 2 + j;
        if (p < pairs) {
          const float x = f[i][2 * j], y = f[i][2 * j + 1];
          f[i][2 * j] = x * cs[p] - y * sn[p];
          f[i][2 * j + 1] = y * cs[p] + x * sn[p];
        }
      }
    }
    if (is_q) store8(a.q + t * a.ld + c, f[i]);
    else if (has_slot) store8(crow + u / a.KD * SL + d, f[i]);
  }
}

// ------------------------------------------------------------------- //
// few queries: one token x up to 16 query heads of one key/value head x one
// key range per workgroup
// ------------------------------------------------------------------- //
struct GroupedDims {
  int H, R, KD, VD, SL, row, tail, max_blocks, n_blocks, n_seqs, window, keep,
      splits, col_groups;
  bool same;
  float out_scale;
  PageRows page;
};

// Each wave walks 32-key tiles of its own: slices go through registers into a
// wave-private LDS tile (the next tile's loads are in flight while this one is
// multiplied), S^T = K Q^T stays in registers and is directly the second
// product's operand, o^T[v][head] += V^T p^T. No barrier until the waves'
// partial sums meet. NL: 16-byte pieces of a tile per lane, NT: 16-column
// value tiles per workgroup.
template <typename T, int NL, int NT>
__global__ __launch_bounds__(256, 2) void grouped_attn_kernel(
    const T* __restrict__ q, long q_t, const T* __restrict__ cache,
    const int* __restrict__ block_table, const int* __restrict__ tok_seq,
    const int* __restrict__ positions, const T* __restrict__ sink,
    T* __restrict__ out, long out_t, float* __restrict__ part_o,
    float* __restrict__ part_ml, GroupedDims d, Score score) {
  constexpr bool PRE = sizeof(T) == 2;
  const int PITCH = d.SL + 8, QP = d.KD + 8;
  const int nw = blockDim.x >> 6;
  extern __shared__ __align__(16) char smem[];
  __shared__ float stat[4][16][2];
  __shared__ __align__(16) float kscale[4][32];
  T* qs = (T*)smem;  // [16][QP]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  T* tile = qs + 16 * QP + wave * 32 * PITCH;  // [32][PITCH]
  const int r16 = lane & 15, g = lane >> 4, ko = g * 8;
  const int t = blockIdx.x;
  const int hc = (d.R + 15) / 16;
  const int hk = blockIdx.y / hc, hr = blockIdx.y % hc * 16;
  const int h0 = hk * d.R + hr, nh = min(16, d.R - hr);
  const int split = blockIdx.z / d.col_groups;
  const int c_base = (blockIdx.z % d.col_groups) * (NT * 16);
  const int cols = min(NT * 16, d.VD - c_base);

  const int bs = d.page.tokens, pool = d.page.pool;
  const int pos = min(max(positions[t], 0), d.max_blocks * bs - 1);
  const int* btab = block_table +
                    (long)min(max(tok_seq[t], 0), d.n_seqs - 1) * d.max_blocks;
  const Visible vis = visible_keys(pos, d.window, d.keep, pool);
  const int n_tiles = (vis.n + 31) / 32;
  const int stride = d.splits * nw;
  int j = split * nw + wave;

  // cached row of key `lane & 31` of a tile; behind the last key, that key's
  auto row_of = [&](int jt) {
    const int i = min(jt * 32 + (lane & 31), vis.n - 1);
    const bool mean = pool > 0 && i < vis.kf;
    const int key = mean ? i * pool + pool - 1 : vis.position(i);
    const int blk = min(max(btab[key / bs], 0), d.n_blocks - 1);
    return mean ? d.page.pooled(blk, key % bs) : d.page.token(blk, key % bs);
  };
  // piece p of a tile: row p / row8, columns 8 * (p % row8)
  const int row8 = d.SL / 8, pieces = 32 * row8;
  int place[PRE ? NL : 1];  // row << 16 | column
  if (PRE) {
#pragma unroll
    for (int i = 0; i < (PRE ? NL : 1); ++i) {
      const int p = min(lane + i * 64, pieces - 1);
      place[i] = (p / row8) << 16 | (p % row8) * 8;
    }
  }
  const T* slice = cache + hk * d.SL;
  uint32x4 pre[PRE ? NL : 1];
  float pre_scale = 1.f;
  auto load = [&](int rows) {
    if (PRE) {
#pragma unroll
      for (int i = 0; i < (PRE ? NL : 1); ++i) {
        const long r = __shfl(rows, place[i] >> 16, 64);
        pre[i] = *reinterpret_cast<const uint32x4*>(
            slice + r * d.row + (place[i] & 0xffff));
      }
    }
    if (d.same)
      pre_scale = reinterpret_cast<const float*>(
          cache + (long)rows * d.row + d.tail)[hk];
  };
  auto store = [&](int rows) {
    if (PRE) {
      // the last pieces are written twice, with the same contents
#pragma unroll
      for (int i = 0; i < (PRE ? NL : 1); ++i)
        *reinterpret_cast<uint32x4*>(
            tile + (place[i] >> 16) * PITCH + (place[i] & 0xffff)) = pre[i];
    }
    for (int p = lane + (PRE ? NL * 64 : 0); p < pieces; p += 64) {
      const int k = p / row8, c = (p % row8) * 8;
      const long r = __shfl(rows, k, 64);
      copy8(tile + k * PITCH + c, slice + r * d.row + c);
    }
    if (d.same && lane < 32) kscale[wave][lane] = pre_scale;
  };

  int rows = row_of(j), rows_n = row_of(j + stride);
  if (j < n_tiles) load(rows);
  const int q8 = d.KD / 8;
  for (int i = tid; i < 16 * q8; i += blockDim.x) {
    const int r = i / q8, c = (i % q8) * 8;
    if (r < nh) copy8(qs + r * QP + c, q + t * q_t + (h0 + r) * d.KD + c);
    else zero8(qs + r * QP + c);
  }
  __syncthreads();

  float m_run = -INFINITY, l_run = 0.f;  // head r16, this lane group's keys
  lm_f32x4 acc[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) acc[i] = lm_f32x4{0.f, 0.f, 0.f, 0.f};
  const T* vt = tile + (d.same ? 0 : d.KD) + c_base;

  for (; j < n_tiles; j += stride) {
    wave_lds_fence();  // the previous tile has been read
    store(rows);
    rows = rows_n;
    if (j + stride < n_tiles) load(rows);
    rows_n = row_of(j + 2 * stride);
    wave_lds_fence();
    lm_f32x4 s[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll 4
    for (int k = 0; k < d.KD; k += 32) {
      const Frag<T> qf = load_frag(qs + r16 * QP + k + ko);
      s[0] = mma32(load_frag(tile + r16 * PITCH + k + ko), qf, s[0]);
      s[1] = mma32(load_frag(tile + (16 + r16) * PITCH + k + ko), qf, s[1]);
    }
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      if (d.same) {
        const lm_f32x4 ks = *reinterpret_cast<const lm_f32x4*>(
            &kscale[wave][i * 16 + 4 * g]);
        s[i] *= ks;
      }
      if (score.capped) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          s[i][r] = score.out2 * cap_tanh<T>(s[i][r] * score.in);
      } else {
        s[i] *= score.scale2;
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (j * 32 + i * 16 + 4 * g + r >= vis.n) s[i][r] = -INFINITY;
        mx = fmaxf(mx, s[i][r]);
      }
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float m_new = fmaxf(m_run, mx);  // finite: a tile has a key
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
    m_run = m_new;
    l_run *= alpha;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        s[i][r] = __builtin_amdgcn_exp2f(s[i][r] - m_new);
        l_run += s[i][r];
      }
    }
    const Frag<T> pf = frag_of<T>(s[0], s[1]);
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      if (i * 16 < cols)
        acc[i] = mma32(load_frag_rows(vt + i * 16, PITCH), pf, acc[i] * alpha);
    }
  }

  // the wave's own tile region holds its sums
  meet_waves<NT>(
      acc, m_run, l_run, cols, nh, stat, (float*)(qs + 16 * QP),
      32 * PITCH * (int)sizeof(T) / 4,
      [&](int r, int c, const lm_f32x4& o, float m, float l) {
        const int h = h0 + r;
        if (d.splits > 1) {
          const long pi = ((long)t * d.H + h) * d.splits + split;
          const float v[4] = {o[0], o[1], o[2], o[3]};
          store4(part_o + pi * d.VD + c_base + c, v);
          if (c == 0 && c_base == 0) {
            part_ml[2 * pi] = m;
            part_ml[2 * pi + 1] = l;
          }
        } else {
          const float inv =
              d.out_scale *
              over_weights(m, l,
                           sink ? to_f32(sink[h]) * LM_LOG2E : -INFINITY);
          const float v[4] = {o[0] * inv, o[1] * inv, o[2] * inv, o[3] * inv};
          store4(out + t * out_t + h * d.VD + c_base + c, v);
        }
      });
}

// ------------------------------------------------------------------- //
// means of whole blocks: a wave for 512 columns of the blocks that `per` tokens
// may end
// ------------------------------------------------------------------- //
template <typename T>
__global__ __launch_bounds__(64) void grouped_pool_kernel(
    T* cache, const int* __restrict__ block_table,
    const int* __restrict__ tok_seq, const int* __restrict__ positions,
    int row, int max_blocks, int n_blocks, int n_seqs, PageRows page, int per,
    int n_tok) {
  const int c = (blockIdx.y * 64 + threadIdx.x) * 8;
  const int end = min((int)(blockIdx.x + 1) * per, n_tok);
  for (int t = blockIdx.x * per; t < end; ++t) {
    const int pos = positions[t];
    if (pos < 0 || (pos + 1) % page.pool || pos >= max_blocks * page.tokens ||
        c >= row)
      continue;
    const int* btab =
        block_table + (long)min(max(tok_seq[t], 0), n_seqs - 1) * max_blocks;
    auto page_of = [&](int p) {
      return min(max(btab[p / page.tokens], 0), n_blocks - 1);
    };
    const float inv = 1.f / (float)page.pool;
    T* dst = cache +
             (long)page.pooled(page_of(pos), pos % page.tokens) * row;
    float sum[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
    for (int p = pos + 1 - page.pool; p <= pos; ++p) {
      float f[8];
      load8<T>(cache + (long)page.token(page_of(p), p % page.tokens) * row + c,
               f);
#pragma unroll
      for (int e = 0; e < 8; ++e) sum[e] += f[e];
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) sum[e] *= inv;
    store8(dst + c, sum);
  }
}

}  // namespace

// z [T, cols] holds q at column 0, k at k_at, v at v_at (-1: values are keys);
// bias [cols] is added; q is finished in place, keys and values go to the
// cache rows of `slots`
void lm_grouped_prep(torch::Tensor z, long k_at, long v_at,
                     torch::Tensor positions, torch::Tensor slots,
                     c10::optional<torch::Tensor> inv_freq, double gain,
                     long H, long G, long KD, long VD, long dim,
                     c10::optional<torch::Tensor> q_norm,
                     c10::optional<torch::Tensor> k_norm, double eps,
                     c10::optional<torch::Tensor> first, double lam,
                     torch::Tensor cache, c10::optional<torch::Tensor> bias,
                     bool whole, long pool) {
  LM_CHECK_I32(positions);
  LM_CHECK_I32(slots);
  LM_CHECK_CONTIG(cache);
  const long T = positions.numel();
  const auto type = z.scalar_type();
  const bool same = v_at < 0;
  const long SL = same ? KD : KD + VD, row = cache.size(2);
  TORCH_CHECK(slots.numel() == T && G >= 1 && H % G == 0);
  TORCH_CHECK(KD % 32 == 0 && VD % 32 == 0 && KD <= 512 && VD <= 512 &&
              dim >= 1 && dim <= KD);
  lm_check_rows(z, T, z.size(1), type);
  TORCH_CHECK(H * KD <= k_at && k_at % 8 == 0 && k_at + G * KD <= z.size(1));
  TORCH_CHECK(same || (v_at % 8 == 0 && v_at >= k_at + G * KD &&
                       v_at + G * VD <= z.size(1)));
  TORCH_CHECK(cache.dim() == 3 && cache.scalar_type() == type &&
              row % 8 == 0 && row >= G * SL);
  if (same)  // a factor per key instead of normed, rotated keys
    TORCH_CHECK(!inv_freq && !first && row - G * SL >= 2 * G,
                "lm_grouped_prep: values are keys");
  for (const auto* w : {&q_norm, &k_norm})
    if (w->has_value())
      TORCH_CHECK((*w)->is_cuda() && (*w)->is_contiguous() &&
                  (*w)->numel() ==
                      KD * (!whole ? 1 : w == &q_norm ? H : G) &&
                  (*w)->scalar_type() == type);
  TORCH_CHECK(!whole || (q_norm && k_norm && !same));
  if (bias)
    TORCH_CHECK(bias->is_cuda() && bias->is_contiguous() && !same &&
                bias->numel() >= v_at + G * VD &&
                bias->scalar_type() == type);
  if (first) lm_check_rows(*first, T, G * VD, type);
  Rot rot{nullptr, 0, 0, 1.f};
  if (inv_freq) rot = make_rot(*inv_freq, gain, false, KD);
  if (T == 0) return;
  int lph = 4;
  while (lph * 8 < std::max(KD, same ? KD : VD)) lph *= 2;
  // few tokens: a workgroup for each, else a wave
  const int per_wg = T <= 1024 ? 1 : 4;
  const long total = (H + G) * KD + G * VD;
  TORCH_CHECK(!whole || (k_at == H * KD && v_at == k_at + G * KD &&
                         total <= 256 * 16 * 8),
              "lm_grouped_prep: norm over ", total, " columns");
#define LM_GPW(NV, TPT)                                                     \
  hipLaunchKernelGGL((grouped_prep_whole_kernel<scalar_t, NV, TPT>),        \
                     dim3((T + 256 / TPT - 1) / (256 / TPT)), dim3(256), lds, \
                     cmls::current_stream(), a, positions.data_ptr<int>(),  \
                     slots.data_ptr<int>(), rot, (int)T)
  LM_DISPATCH(z, "lm_grouped_prep", [&] {
    GroupedPrep<scalar_t> a{};
    a.q = (scalar_t*)z.data_ptr();
    a.k = a.q + k_at;
    a.v = same ? nullptr : a.q + v_at;
    a.ld = z.stride(0);
    if (first) {
      a.first = (const scalar_t*)first->data_ptr();
      a.ld_first = first->stride(0);
      a.lam = (float)lam;
    }
    a.qn = q_norm ? (const scalar_t*)q_norm->data_ptr() : nullptr;
    a.kn = k_norm ? (const scalar_t*)k_norm->data_ptr() : nullptr;
    if (bias) {
      a.qb = (const scalar_t*)bias->data_ptr();
      a.kb = a.qb + k_at;
      a.vb = a.qb + v_at;
    }
    a.page = page_rows(cache.size(1), pool);
    a.cache = (scalar_t*)cache.data_ptr();
    a.n_slots = (long)cache.size(0) * a.page.tokens;
    a.H = (int)H;
    a.G = (int)G;
    a.KD = (int)KD;
    a.VD = (int)VD;
    a.dim = (int)dim;
    a.row = (int)row;
    a.eps = (float)eps;
    if (whole) {
      const size_t lds = std::max(1, 4 * 2 * rot.pairs) * 4;
      // a wave per token where its vectors fit and there are enough tokens
      if (total <= 64 * 8 * 8 && T > 1024) LM_GPW(8, 64);
      else if (total <= 256 * 4 * 8) LM_GPW(4, 256);
      else LM_GPW(16, 256);
      return;
    }
    hipLaunchKernelGGL((grouped_prep_kernel<scalar_t>),
                       dim3((T + per_wg - 1) / per_wg), dim3(256),
                       std::max(1, per_wg * 2 * rot.pairs) * 4,
                       cmls::current_stream(), a, positions.data_ptr<int>(),
                       slots.data_ptr<int>(), rot, (int)T, per_wg, lph);
  });
#undef LM_GPW
  LM_LAUNCHED();
}

// the means of the blocks that the given tokens end, into their pages
void lm_grouped_pool(torch::Tensor cache, torch::Tensor block_table,
                     torch::Tensor tok_seq, torch::Tensor positions,
                     long pool) {
  LM_CHECK_CONTIG(cache);
  LM_CHECK_I32(block_table);
  LM_CHECK_I32(tok_seq);
  LM_CHECK_I32(positions);
  const long T = positions.numel(), row = cache.size(2);
  TORCH_CHECK(pool >= 1 && cache.dim() == 3 && row % 8 == 0 &&
              tok_seq.numel() == T && block_table.dim() == 2);
  if (T == 0) return;
  TORCH_CHECK(block_table.numel() > 0);
  const PageRows page = page_rows(cache.size(1), pool);
  // decoded tokens may all end one; of a portion's tokens every pool-th does
  const int per = T <= 1024 ? 1 : (int)std::min<long>(pool, 16);
  LM_DISPATCH(cache, "lm_grouped_pool", [&] {
    hipLaunchKernelGGL((grouped_pool_kernel<scalar_t>),
                       dim3((T + per - 1) / per, (row + 511) / 512), dim3(64),
                       0, cmls::current_stream(),
                       (scalar_t*)cache.data_ptr(),
                       block_table.data_ptr<int>(), tok_seq.data_ptr<int>(),
                       positions.data_ptr<int>(), (int)row,
                       (int)block_table.size(1), (int)cache.size(0),
                       (int)block_table.size(0), page, per, (int)T);
  });
  LM_LAUNCHED();
}

// tokens [0, n) of q [T, H * KD] (row stride free) attend to their sequences'
// cache rows -> out [T, H * VD] (row stride free), times out_scale
void lm_grouped_attention(torch::Tensor q, torch::Tensor cache,
                          torch::Tensor block_table, torch::Tensor tok_seq,
                          torch::Tensor positions,
                          c10::optional<torch::Tensor> sink,
                          torch::Tensor out, long n, long H, long G, long KD,
                          long VD, bool same, long window, long keep,
                          long pool, double scale, double cap,
                          double out_scale, long max_keys) {
  LM_CHECK_CONTIG(cache);
  LM_CHECK_I32(block_table);
  LM_CHECK_I32(tok_seq);
  LM_CHECK_I32(positions);
  const auto type = q.scalar_type();
  TORCH_CHECK(G >= 1 && H % G == 0 && KD % 32 == 0 && VD % 32 == 0);
  const long SL = same ? KD : KD + VD;
  TORCH_CHECK(n >= 0 && n <= q.size(0) && out.size(0) == q.size(0));
  lm_check_rows(q, q.size(0), q.size(1), type);
  TORCH_CHECK(q.size(1) >= H * KD && (!same || KD == VD));
  lm_check_rows(out, q.size(0), H * VD, type);
  TORCH_CHECK(cache.dim() == 3 && cache.scalar_type() == type &&
              cache.size(2) % 8 == 0 && cache.size(2) >= G * SL &&
              SL < 65536);
  TORCH_CHECK(!same || cache.size(2) - G * SL >= 2 * G);
  TORCH_CHECK(block_table.dim() == 2 && tok_seq.numel() >= n &&
              positions.numel() >= n);
  TORCH_CHECK(window >= 0 && keep >= 0 &&
              ((keep == 0 && pool == 0) || window > 0) &&
              (keep == 0 || pool == 0) && (pool == 0 || !same));
  if (sink) {
    LM_CHECK_CONTIG(*sink);
    TORCH_CHECK(sink->numel() == H && sink->scalar_type() == type);
  }
  if (n == 0) return;
  TORCH_CHECK(block_table.numel() > 0);
  const int tiles = (int)(VD / 16);
  const int nt = tiles <= 2 ? 2 : tiles <= 4 ? 4 : tiles <= 8 ? 8 : 16;
  const int cgroups = (tiles + nt - 1) / nt;
  const int isz = q.element_size();
  auto lds = [&](int nw) {
    return (16 * (KD + 8) + 32 * nw * (SL + 8)) * isz;
  };
  int nw = 4;
  while (nw > 1 && lds(nw) > 156 * 1024) --nw;
  TORCH_CHECK(lds(nw) <= 156 * 1024, "lm_grouped_attention: head of ", SL,
              " elements does not fit LDS");
  const int hg = (int)(G * ((H / G + 15) / 16));
  // fill 256 CUs as far as there are 32-key tiles for every wave
  const long keys =
      window > 0 ? std::min(window + keep + (pool ? max_keys / pool : 0),
                            max_keys)
                 : max_keys;
  const long per_cu = std::min<long>(2, 156 * 1024 / lds(nw));
  long splits = 256 * per_cu / std::max<long>(1, (long)n * hg * cgroups);
  splits = std::max<long>(1, std::min(splits,
                                      (keys + 32 * nw - 1) / (32 * nw)));
  TORCH_CHECK(hg <= 65535 && splits * cgroups <= 65535);
  torch::Tensor po, pml;
  if (splits > 1) {
    auto f32 = q.options().dtype(at::kFloat);
    po = torch::empty({n, H, splits, VD}, f32);
    pml = torch::empty({n, H, splits, 2}, f32);
  }
  GroupedDims d{};
  d.H = (int)H;
  d.R = (int)(H / G);
  d.KD = (int)KD;
  d.VD = (int)VD;
  d.SL = (int)SL;
  d.row = (int)cache.size(2);
  d.tail = (int)(G * SL);
  d.page = page_rows(cache.size(1), pool);
  d.max_blocks = (int)block_table.size(1);
  d.n_blocks = (int)cache.size(0);
  d.n_seqs = (int)block_table.size(0);
  d.window = (int)window;
  d.keep = (int)keep;
  d.splits = (int)splits;
  d.col_groups = cgroups;
  d.same = same;
  d.out_scale = (float)out_scale;
  const Score score = make_score(scale, cap);
  hipStream_t st = cmls::current_stream();
#define LM_GA(NL, NT)                                                        \
  do {                                                                       \
    const int bytes = (int)lds(nw);                                          \
    auto* fn = &grouped_attn_kernel<scalar_t, NL, NT>;                       \
    HIP_CHECK(hipFuncSetAttribute(                                           \
        reinterpret_cast<const void*>(fn),                                   \
        hipFuncAttributeMaxDynamicSharedMemorySize, bytes));                 \
    hipLaunchKernelGGL(fn, dim3(n, hg, splits * cgroups), dim3(64 * nw),     \
                       bytes, st, (const scalar_t*)q.data_ptr(),             \
                       q.stride(0), (const scalar_t*)cache.data_ptr(),       \
                       block_table.data_ptr<int>(), tok_seq.data_ptr<int>(), \
                       positions.data_ptr<int>(),                            \
                       sink ? (const scalar_t*)sink->data_ptr() : nullptr,   \
                       (scalar_t*)out.data_ptr(), out.stride(0),             \
                       splits > 1 ? po.data_ptr<float>() : nullptr,          \
                       splits > 1 ? pml.data_ptr<float>() : nullptr, d,      \
                       score);                                               \
  } while (0)
#define LM_GA_T(NL)                                                          \
  do {                                                                       \
    if (nt == 2) LM_GA(NL, 2);                                               \
    else if (nt == 4) LM_GA(NL, 4);                                          \
    else if (nt == 8) LM_GA(NL, 8);                                          \
    else LM_GA(NL, 16);                                                      \
  } while (0)
  LM_DISPATCH(q, "lm_grouped_attention", [&] {
    const long nl = SL / 16;  // 32 rows of SL / 8 pieces over 64 lanes
    if (sizeof(scalar_t) == 4) LM_GA_T(1);
    else if (nl <= 4) LM_GA_T(4);
    else if (nl <= 8) LM_GA_T(8);
    else if (nl <= 12) LM_GA_T(12);
    else if (nl <= 16) LM_GA_T(16);
    else if (nl <= 24) LM_GA_T(24);
    else LM_GA_T(32);
    if (splits > 1)
      hipLaunchKernelGGL((combine_ranges_kernel<scalar_t>), dim3(n * H),
                         dim3(128), 0, st, po.data_ptr<float>(),
                         pml.data_ptr<float>(),
                         sink ? (const scalar_t*)sink->data_ptr() : nullptr,
                         (scalar_t*)out.data_ptr(), out.stride(0),
                         (int)splits, (int)H, (int)VD, (float)out_scale);
  });
#undef LM_GA_T
#undef LM_GA
  LM_LAUNCHED();
}
