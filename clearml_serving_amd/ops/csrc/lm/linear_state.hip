// Linear recurrences with one decay per head behind a short convolution: the
// gated delta rule and the state-space recurrence. Per token and head, with
// q, k of the head's group and a float state S [key][value]:
//
//   g = -exp(a_log) softplus(a + dt_bias)
//   DELTA:  q, k unit vectors, q times dim^-1/2;  b = sigmoid(zb)
//           S <- e^g S;  u = b (v - S^T k);  S <- S + k u^T;  o = S^T q
//           out = o / rms(o) * norm * silu(gate)
//   else:   d = softplus(a + dt_bias)
//           S <- e^g S + k (d v)^T;  o = S^T q + skip v
//           out = p / rms(p) * norm, p = o silu(gate), in equal parts
//
// Rows of z: [q | k | v | gate | a | b], of which q, k and v pass a causal
// convolution over time and SiLU.
//
// Single tokens: one fused kernel, a workgroup per token and head. Portions:
// the convolution, then a kernel that walks a sequence in chunks of 32 tokens
// with matrix products in 32-bit. With G the sum of g from a chunk's start on,
// k, q, v the chunk's rows and S the state in front of it,
//
//   (1 + A) U = b (V - e^G K S),   A[t][s] = b_t e^(G_t - G_s) k_t.k_s, s < t
//   O = e^G Q S + M U,             M[t][s] = e^(G_t - G_s) q_t.k_s, s <= t
//   S <- e^G_end S + sum_t e^(G_end - G_t) k_t u_t^T
//
// and U = d V without DELTA. The columns of S do not depend on each other: a
// wave keeps 16 of them in registers, all keys, as results of 16x16 products
// that are at once operands of the next (the order of an MFMA's inner index is
// free), so S, U and what leads to them never leave registers. K and Q are read
// from LDS; K K^T and Q K^T are shared out among the waves; the diagonal 16x16
// blocks of 1 + A are inverted, the rest is substituted block by block.
// Exponents are sums of decays of like sign, never differences across a block.
//
// Few long portions would leave most CUs idle, so these are cut into segments.
// A segment turns the state in front of it into P S + Q: the same kernel makes P
// from the identity without values and Q from zero (without DELTA P is one
// number), a chain over the segments gives the state in front of each
// (state_chain_kernel), and the segments are walked from there.
//
// State in memory: [slot][head][value][key]; the convolution's past inputs as a
// ring [slot][taps][channels] indexed by position, one entry more than it looks
// back, so a token's own entry is never one that it reads. Neither is ever
// cleared: position 0 starts from zero.
#include "lm_attn.h"

namespace {

constexpr int MAX_TAPS = 8;

// eight elements as they are
template <typename T> struct alignas(16) Raw8 {
  T v[8];
};

template <typename T>
struct StateArgs {
  const T* z;        // rows of ld
  long ld;
  int k_at, v_at, gate_at, a_at, b_at, channels;
  const T *conv, *conv_b;           // [taps, channels], [channels] or null
  const T *a_log, *dt_bias, *skip;  // [heads]; skip without DELTA only
  const T* norm;                    // [heads * VP]
  float* state;      // [slots, heads, VP, KP]
  T* ring;           // [slots, taps, channels]
  T* u;              // convolved rows of the portions, [rows + CH, channels]
  float* decay;      // [tiles, heads, 2, DECAY] of the portions' chunks
  T* y;              // o of all tokens, [T, heads * VP]
  T* out;            // rows of ld_out
  long ld_out;
  const int *positions, *slots, *tiles, *seqs;
  int n_single, n_seq, n_state, n_tok, heads, groups, KP, VP, dim, vdim, taps,
      parts;
  float eps;
  // portions are walked in segments of `seg` tiles, 0: whole
  int seg, n_seg;   // n_seg: bound on all portions' segments
  float *P, *Q;     // [n_seg, heads, KP, KP] and [n_seg, heads, VP, KP]
};

__device__ __forceinline__ int segments_of(const int* portion, int seg) {
  return (portion[1] + seg - 1) / seg;
}

template <typename T>
__device__ __forceinline__ float silu_f(float z) {
  return z * sigmoid_f(z);
}
template <> __device__ __forceinline__ float silu_f<float>(float z) {
  return z / (1.f + expf(-z));
}

// log decay and step of a head for its raw input
__device__ __forceinline__ void decay_of(float a, float a_log, float dt_bias,
                                         float* g, float* step) {
  *step = softplus_f(a + dt_bias);
  *g = -expf(a_log) * *step;
}

__device__ __forceinline__ float sum8(float v) {  // lanes that share lane >> 3
  v += __shfl_xor(v, 1, 64);
  v += __shfl_xor(v, 2, 64);
  return v + __shfl_xor(v, 4, 64);
}

// ------------------------------------------------------------------- //
// convolution and SiLU of the portions' tokens
// ------------------------------------------------------------------- //
constexpr int TILE = 64;              // tokens of the host's tiles
constexpr int CH = 32, NB = CH / 16;  // tokens of a chunk, its blocks

struct ChunkDecay {
  float in[CH];    // e^(G_t)
  float out[CH];   // e^(G_end - G_t)
  float step[CH];  // b_t or d_t
  float run[CH];   // sum of g from the block's start to t
  float rest[CH];  // sum of g behind t to the block's end
  float total;     // e^(G_end)
  float pad[3];
};
constexpr int DECAY = sizeof(ChunkDecay) / 4;

// the decays of a tile's two chunks, a wave per head
template <typename T, bool DELTA>
__device__ __forceinline__ void tile_decays(const StateArgs<T>& p, int tile,
                                            int h) {
  const int t0 = p.tiles[tile * 5], len = p.tiles[tile * 5 + 1];
  const int lane = threadIdx.x & 63, r16 = lane & 15;
  float gt = 0.f, step = 0.f;
  if (lane < len) {
    const T* row = p.z + (long)(t0 + lane) * p.ld;
    decay_of(to_f32(row[p.a_at + h]), to_f32(p.a_log[h]),
             to_f32(p.dt_bias[h]), &gt, &step);
    if (DELTA) step = 1.f / (1.f + expf(-to_f32(row[p.b_at + h])));
  }
  float run = gt, rest = gt;
#pragma unroll
  for (int d = 1; d < 16; d <<= 1) {
    const float a = __shfl_up(run, d, 16), b = __shfl_down(rest, d, 16);
    if (r16 >= d) run += a;
    if (r16 + d < 16) rest += b;
  }
  const int half = lane & 32;
  const float first = __shfl(run, half + 15, 64);
  const float second = __shfl(run, half + 31, 64);
  const float behind = __shfl_down(rest, 1, 16);
  rest = r16 == 15 ? 0.f : behind;
  ChunkDecay* d = (ChunkDecay*)p.decay +
                  ((long)tile * p.heads + h) * 2 + (half ? 1 : 0);
  const int t = lane & 31;
  d->run[t] = run;
  d->rest[t] = rest;
  d->step[t] = step;
  d->in[t] = expf(t < 16 ? run : first + run);
  d->out[t] = expf(t < 16 ? rest + second : rest);
  if (t == 0) d->total = expf(first + second);
}

// A thread takes 8 channels of up to 8 tokens; TAPS >= taps. The grid's last
// rows make the chunks' decays.
template <typename T, int TAPS, bool DELTA>
__global__ __launch_bounds__(256) void state_conv_kernel(StateArgs<T> p,
                                                         int n_conv) {
  if ((int)blockIdx.y >= n_conv) {
    const int h = (blockIdx.y - n_conv) * 4 + (threadIdx.x >> 6);
    if (h < p.heads) tile_decays<T, DELTA>(p, blockIdx.x, h);
    return;
  }
  const int* td = p.tiles + blockIdx.x * 5;
  const int t0 = td[0], len = td[1], p0 = td[2], slot = td[3], into = td[4];
  const int c = (blockIdx.y * 32 + (threadIdx.x & 31)) * 8;
  if (c >= p.channels) return;
  const bool has_state = slot >= 0 && slot < p.n_state;
  float w[TAPS][8], bias[8];
#pragma unroll
  for (int d = 0; d < TAPS; ++d) {  // d tokens back
#pragma unroll
    for (int e = 0; e < 8; ++e) w[d][e] = 0.f;
    if (d < p.taps)
      load8<T>(p.conv + (long)(p.taps - 1 - d) * p.channels + c, w[d]);
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) bias[e] = 0.f;
  if (p.conv_b) load8<T>(p.conv_b + c, bias);
  for (int r0 = (threadIdx.x >> 5) * 8; r0 < len; r0 += 64) {
    float past[TAPS][8];  // past[d]: the input d + 1 tokens back
#pragma unroll
    for (int d = 0; d < TAPS; ++d) {
#pragma unroll
      for (int e = 0; e < 8; ++e) past[d][e] = 0.f;
      const int back = d + 1, pos = p0 + r0 - back;
      if (back < p.taps && pos >= 0) {
        if (back <= r0 + into)
          load8<T>(p.z + (long)(t0 + r0 - back) * p.ld + c, past[d]);
        else if (has_state)
          load8<T>(p.ring +
                       ((long)slot * p.taps + pos % p.taps) * p.channels + c,
                   past[d]);
      }
    }
    const int n = min(8, len - r0);
    Raw8<T> raw[8];
#pragma unroll
    for (int i = 0; i < 8; ++i)
      raw[i] = *reinterpret_cast<const Raw8<T>*>(
          p.z + (long)(t0 + r0 + min(i, n - 1)) * p.ld + c);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      float x[8], f[8];
      load8<T>(raw[i].v, x);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        f[e] = bias[e] + w[0][e] * x[e];
#pragma unroll
        for (int d = 1; d < TAPS; ++d) f[e] += w[d][e] * past[d - 1][e];
        f[e] = silu_f<T>(f[e]);
#pragma unroll
        for (int d = TAPS - 1; d > 0; --d) past[d][e] = past[d - 1][e];
        past[0][e] = x[e];
      }
      if (i < n)
        store8(p.u + (long)(t0 + r0 + i - p.n_single) * p.channels + c, f);
    }
  }
}

// ------------------------------------------------------------------- //
// portions in chunks
// ------------------------------------------------------------------- //
// sum over N neighbouring lanes, in all of them (DPP within 16 lanes)
template <int N> __device__ __forceinline__ float sum_lanes(float v) {
#define LM_DPP_ADD(CTRL)                                      \
  v += __int_as_float(__builtin_amdgcn_update_dpp(            \
      0, __float_as_int(v), CTRL, 0xf, 0xf, true))
  LM_DPP_ADD(0xB1);                       // quad_perm 1 0 3 2
  LM_DPP_ADD(0x4E);                       // quad_perm 2 3 0 1
  if (N >= 8) LM_DPP_ADD(0x141);          // row_half_mirror
  if (N >= 16) LM_DPP_ADD(0x140);         // row_mirror
#undef LM_DPP_ADD
  if (N >= 32) v += __shfl_xor(v, 16, 64);
  return v;
}

// a[16 rows][K] . b[16 rows][K]^T, rows of `pitch` in LDS
__device__ __forceinline__ lm_f32x4 dot_rows(const float* a, const float* b,
                                             int pitch, int K) {
  const int lane = threadIdx.x & 63, at = (lane & 15) * pitch + 4 * (lane >> 4);
  lm_f32x4 c0 = {0.f, 0.f, 0.f, 0.f}, c1 = c0;
#pragma unroll
  for (int k = 0; k < K; k += 32) {
    const lm_f32x4 x0 = *reinterpret_cast<const lm_f32x4*>(a + at + k);
    const lm_f32x4 y0 = *reinterpret_cast<const lm_f32x4*>(b + at + k);
    const lm_f32x4 x1 = *reinterpret_cast<const lm_f32x4*>(a + at + k + 16);
    const lm_f32x4 y1 = *reinterpret_cast<const lm_f32x4*>(b + at + k + 16);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      c0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x0[r], y0[r], c0, 0, 0, 0);
      c1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x1[r], y1[r], c1, 0, 0, 0);
    }
  }
  return c0 + c1;
}
// c + a b: a rows in LDS (row = lane & 15), b a result in registers
__device__ __forceinline__ lm_f32x4 mul_tile(const float* a, int pitch,
                                             const lm_f32x4& b, lm_f32x4 c) {
  const int lane = threadIdx.x & 63;
  const lm_f32x4 x = *reinterpret_cast<const lm_f32x4*>(
      a + (lane & 15) * pitch + 4 * (lane >> 4));
#pragma unroll
  for (int r = 0; r < 4; ++r)
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(x[r], b[r], c, 0, 0, 0);
  return c;
}

// The elements of two 16-token blocks' products: rows t of block bi, columns s
// of block bj, times the decay between s and t
__device__ __forceinline__ lm_f32x4 decayed(lm_f32x4 c, const ChunkDecay& d,
                                            int bi, int bj) {
  const int lane = threadIdx.x & 63, s = bj * 16 + (lane & 15);
  const lm_f32x4 run =
      *reinterpret_cast<const lm_f32x4*>(d.run + bi * 16 + 4 * (lane >> 4));
  // in one block the difference of two sums of it
  const float from_s = bi == bj ? -d.run[s] : d.rest[s];
#pragma unroll
  for (int r = 0; r < 4; ++r) c[r] *= exp_f(fminf(run[r] + from_s, 0.f));
  return c;
}

// D: 32-channel blocks of a key. Grid (heads * slices of 64 values,
// sequences). Four waves keep the state, 16 values each; four more prepare the
// next chunk meanwhile: they stage its rows while the first ones multiply this
// chunk's with the state, and make its A and M while the others finish. COMPOSE:
// P and Q of a segment instead of outputs, values behind the columns of P.
constexpr int NW = 4, NTH = NW * 64;
template <typename T, int D, bool DELTA, bool COMPOSE>
__global__ __launch_bounds__(2 * NTH, 2)
void state_chunk_kernel(StateArgs<T> p) {
  constexpr int KP = D * 32, PITCH = KP + 4, AP = CH + 4;
  constexpr int AM = (DELTA ? 2 : 1) * CH * AP;  // -A and inverses, M
  // staging: LPR lanes take a row, RPI rows at a time
  constexpr int LPR = D <= 1 ? 4 : D <= 2 ? 8 : D <= 4 ? 16 : 32;
  constexpr int RPI = NTH / LPR, NI = 2 * CH / RPI;
  static_assert(NI * RPI == 2 * CH, "rows");
  extern __shared__ __align__(16) float sm[];
  float* sk = sm;                   // 2 x [K rows | Q rows]
  float* sam = sm + 4 * CH * PITCH; // 2 x [M | A], [CH][AP] each
  float* sd = sam + 2 * AM;         // 2 x DECAY
  const int lane = threadIdx.x & 63, wave = uniform_wave() % NW;
  const int tid = wave * 64 + lane;  // within the four waves
  const bool keeps = uniform_wave() < NW;
  const int r16 = lane & 15, g = lane >> 4;
  const int h = blockIdx.x % p.heads, slice = blockIdx.x / p.heads;
  // long sequences first: they are the last of the list
  int seq = p.n_seq - 1 - (int)blockIdx.y, part = 0;
  if (p.seg) {  // segment `part` of a portion
    part = blockIdx.y;
    seq = 0;
    while (seq < p.n_seq && part >= segments_of(p.seqs + seq * 6, p.seg))
      part -= segments_of(p.seqs + seq++ * 6, p.seg);
    if (seq == p.n_seq) return;
  }
  const int* sq = p.seqs + seq * 6;
  const bool ends = !p.seg || part + 1 == segments_of(sq, p.seg);
  if (COMPOSE && ends) return;  // nothing follows
  const int skipped = part * p.seg * TILE;
  const int t0 = sq[2] + skipped, p0 = sq[4], slot = sq[5];
  const int len = ends ? sq[3] - skipped : p.seg * TILE;
  const bool has_state = slot >= 0 && slot < p.n_state;
  const int hk = h / (p.heads / p.groups);
  const T* urow = p.u + (long)(t0 - p.n_single) * p.channels;

  if (!keeps) {
    const float* drow =
        p.decay + ((long)(sq[0] + part * p.seg) * p.heads + h) * 2 * DECAY;
    Raw8<T> kq[NI];
    lm_f32x4 dreg = {0.f, 0.f, 0.f, 0.f};
    const int item_row = tid / LPR, item_c = tid % LPR * 8;
    const bool item_in = LPR * 8 == KP || item_c < KP;
    const unsigned item_at = item_row * p.channels + (item_in ? item_c : 0);
    const float q_scale = DELTA ? 1.f / sqrtf((float)p.dim) : 1.f;
    auto load = [&](int at) {
      // u has CH more rows than there are tokens
      const T* q = urow + (long)at * p.channels + hk * KP;
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        if (RPI > CH) {  // K and Q rows at once
          const bool is_q = item_row >= CH;
          kq[i] = *reinterpret_cast<const Raw8<T>*>(
              q + (long)(item_row % CH) * p.channels + item_c +
              (is_q ? 0 : p.k_at));
        } else {
          const bool is_q = i * RPI >= CH;
          if (COMPOSE && is_q) continue;
          kq[i] = *reinterpret_cast<const Raw8<T>*>(
              q + (is_q ? 0 : p.k_at) + (i * RPI % CH) * p.channels + item_at);
        }
      }
      if (tid < DECAY / 4)
        dreg = reinterpret_cast<const lm_f32x4*>(
            drow + ((long)(at / TILE) * p.heads * 2 + at / CH % 2) *
                       DECAY)[tid];
    };
    auto store = [&](int at, int buf) {
      const int nt = min(CH, len - at);
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        if (COMPOSE && RPI <= CH && i * RPI >= CH) continue;  // no Q rows
        const int row = i * RPI + item_row;
        const bool live = row % CH < nt && item_in;
        float f = 1.f, x[8];
        load8<T>(kq[i].v, x);
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = live ? x[e] : 0.f;
        if (DELTA) {
          float ss = 0.f;
#pragma unroll
          for (int e = 0; e < 8; ++e) ss += x[e] * x[e];
          ss = sum_lanes<LPR>(ss);
          f = __builtin_amdgcn_rsqf(ss + 1e-6f);
          if (row >= CH) f *= q_scale;
        }
        if (item_in) {
#pragma unroll
          for (int e = 0; e < 8; ++e) x[e] *= f;
          store8(sk + (buf * 2 * CH + row) * PITCH + item_c, x);
        }
      }
      if (tid < DECAY / 4)
        reinterpret_cast<lm_f32x4*>(sd + buf * DECAY)[tid] = dreg;
    };
    // the lower 16x16 blocks of K K^T and Q K^T: waves 0 and 1 the diagonal
    // ones of K K^T, which they also invert
    auto products = [&](int buf) {
      const float* K = sk + buf * 2 * CH * PITCH;
      const float* Q = K + CH * PITCH;
      float* sM = sam + buf * AM;
      float* sa = sM + CH * AP;
      const ChunkDecay& d =
          *reinterpret_cast<const ChunkDecay*>(sd + buf * DECAY);
      auto put_m = [&](lm_f32x4 m, int bi, int bj) {
        m = decayed(m, d, bi, bj);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          sM[(bi * 16 + 4 * g + r) * AP + bj * 16 + r16] =
              bi == bj && r16 > 4 * g + r ? 0.f : m[r];
      };
      if (!DELTA) {
        if (!COMPOSE && wave < 3) {
          const int bi = wave > 0, bj = wave == 1;
          put_m(dot_rows(Q + bi * 16 * PITCH, K + bj * 16 * PITCH, PITCH, KP),
                bi, bj);
        }
      } else if (wave < 2) {
        const float* k = K + wave * 16 * PITCH;
        lm_f32x4 c = decayed(dot_rows(k, k, PITCH, KP), d, wave, wave);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          c[r] = r16 < 4 * g + r ? c[r] * -d.step[wave * 16 + 4 * g + r] : 0.f;
        // 1 / (1 + A) by substitution, a lane per column; c holds -A, whose
        // element (i, j) is register i % 4 of lane 16 (i / 4) + j
        float* dst = sa + wave * (16 * AP + 16) + r16;
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          float even = i == r16 ? 1.f : 0.f, odd = 0.f;
#pragma unroll
          for (int j = 0; j < 16; ++j) {
            if (j >= i) continue;
            const float m = __int_as_float(__builtin_amdgcn_readlane(
                __float_as_int(c[i & 3]), 16 * (i >> 2) + j));
            if (j & 1) odd += m * x[j];
            else even += m * x[j];
          }
          x[i] = even + odd;
          if (lane < 16) dst[i * AP] = x[i];
        }
      } else if (wave == 2) {
        lm_f32x4 kk = dot_rows(K + 16 * PITCH, K, PITCH, KP);
        kk = decayed(kk, d, 1, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          sa[(16 + 4 * g + r) * AP + r16] = kk[r] * -d.step[16 + 4 * g + r];
        if (!COMPOSE) put_m(dot_rows(Q + 16 * PITCH, K, PITCH, KP), 1, 0);
      } else if (!COMPOSE) {
        const lm_f32x4 m0 = dot_rows(Q, K, PITCH, KP);
        const lm_f32x4 m1 =
            dot_rows(Q + 16 * PITCH, K + 16 * PITCH, PITCH, KP);
        put_m(m0, 0, 0);
        put_m(m1, 1, 1);
      }
    };
    load(0);
    store(0, 0);
    if (CH < len) load(CH);
    __syncthreads();
    products(0);
    __syncthreads();
    int buf = 0;
    for (int at = CH; at < len; at += CH) {  // at: the next chunk
      buf ^= 1;
      store(at, buf);
      if (at + CH < len) load(at + CH);
      __syncthreads();
      products(buf);
      __syncthreads();
    }
    __syncthreads();  // the last chunk's, where nothing is next
  } else {
    // the wave's columns: values, in COMPOSE behind those of P
    const int c0 = (slice * NW + wave) * 16;
    const bool of_p = COMPOSE && DELTA && c0 < KP;
    const int v0 = COMPOSE && DELTA && !of_p ? c0 - KP : c0;
    const bool active = of_p || v0 < p.VP;  // else nobody uses what it makes
    const int col = active ? v0 + r16 : 0;
    const long unit = (long)blockIdx.y * p.heads + h;
    float* st = p.state + ((long)(has_state ? slot : 0) * p.heads + h) *
                              p.VP * KP;
    const float* from = p.seg ? p.Q + unit * p.VP * KP : st;
    float* to = of_p ? p.P + unit * KP * KP
                     : COMPOSE ? p.Q + unit * p.VP * KP : st;
    from += col * KP + 4 * g;
    to += col * KP + 4 * g;
    lm_f32x4 S[2 * D];  // S[i][r]: key 16 i + 4 g + r, value r16
    if (COMPOSE) {
#pragma unroll
      for (int i = 0; i < 2 * D; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          S[i][r] = of_p && 16 * i + 4 * g + r == col ? 1.f : 0.f;
    } else if (p.seg || (p0 > 0 && has_state)) {
#pragma unroll
      for (int i = 0; i < 2 * D; ++i)
        S[i] = *reinterpret_cast<const lm_f32x4*>(from + 16 * i);
    } else {
#pragma unroll
      for (int i = 0; i < 2 * D; ++i) S[i] = lm_f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const float skip = DELTA ? 0.f : to_f32(p.skip[h]);
    const int ld_y = p.heads * p.VP;
    const unsigned lane_v = 4 * g * p.channels + (of_p ? 0 : col);
    const unsigned lane_y = 4 * g * ld_y + col;
    T vr[NB][4], vn[NB][4];  // values of this chunk and the next
    auto load_values = [&](int at, T (&v)[NB][4]) {
      const T* row = urow + (long)at * p.channels + p.v_at + h * p.VP;
#pragma unroll
      for (int i = 0; i < NB; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          v[i][r] = (row + (16 * i + r) * p.channels)[lane_v];
    };
    load_values(0, vn);
    __syncthreads();
    __syncthreads();
    int buf = 0;
    for (int at = 0; at < len; at += CH, buf ^= 1) {
      const int nt = min(CH, len - at);
#pragma unroll
      for (int i = 0; i < NB; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) vr[i][r] = vn[i][r];
      if (at + CH < len) load_values(at + CH, vn);
      const float* K = sk + buf * 2 * CH * PITCH;
      const float* Q = K + CH * PITCH;
      const float* sM = sam + buf * AM;
      const float* sa = sM + CH * AP;
      const ChunkDecay& d =
          *reinterpret_cast<const ChunkDecay*>(sd + buf * DECAY);
      // products with the state in front of the chunk
      lm_f32x4 R[NB], O[NB];
#pragma unroll
      for (int i = 0; i < NB; ++i) R[i] = O[i] = lm_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < 2 * D; ++k) {
#pragma unroll
        for (int i = 0; i < NB; ++i) {
          if (!COMPOSE)
            O[i] = mul_tile(Q + i * 16 * PITCH + 16 * k, PITCH, S[k], O[i]);
          if (DELTA)
            R[i] = mul_tile(K + i * 16 * PITCH + 16 * k, PITCH, S[k], R[i]);
        }
      }
      __syncthreads();
      lm_f32x4 U[NB];
#pragma unroll
      for (int i = 0; i < NB; ++i) {
        const int tr = 16 * i + 4 * g;
        const lm_f32x4 in = *reinterpret_cast<const lm_f32x4*>(d.in + tr);
        const lm_f32x4 step = *reinterpret_cast<const lm_f32x4*>(d.step + tr);
        lm_f32x4 v;
#pragma unroll
        for (int r = 0; r < 4; ++r)
          v[r] = !of_p && tr + r < nt ? to_f32(vr[i][r]) : 0.f;
        O[i] *= in;
        if (DELTA) {
          lm_f32x4 x = step * (v - in * R[i]);
          if (i == 1) x = mul_tile(sa + 16 * AP, AP, U[0], x);
          U[i] = mul_tile(sa + i * (16 * AP + 16), AP, x,
                          lm_f32x4{0.f, 0.f, 0.f, 0.f});
        } else {
          O[i] += skip * v;
          U[i] = step * v;
        }
      }
      if (!COMPOSE) {
        O[0] = mul_tile(sM, AP, U[0], O[0]);
        O[1] = mul_tile(sM + 16 * AP, AP, U[0], O[1]);
        O[1] = mul_tile(sM + 16 * AP + 16, AP, U[1], O[1]);
      }
      // the state behind the chunk
#pragma unroll
      for (int i = 0; i < NB; ++i)
        U[i] *= *reinterpret_cast<const lm_f32x4*>(d.out + 16 * i + 4 * g);
      const float total = d.total;
#pragma unroll
      for (int k = 0; k < 2 * D; ++k) {
        S[k] *= total;
#pragma unroll
        for (int i = 0; i < NB; ++i) {
          const float* col_k = K + (16 * i + 4 * g) * PITCH + 16 * k + r16;
#pragma unroll
          for (int r = 0; r < 4; ++r)
            S[k] = __builtin_amdgcn_mfma_f32_16x16x4f32(
                col_k[r * PITCH], U[i][r], S[k], 0, 0, 0);
        }
      }
      T* yrow = p.y + (long)(t0 + at) * ld_y + h * p.VP;
      if (COMPOSE) {
      } else if (active && nt == CH) {
#pragma unroll
        for (int i = 0; i < NB; ++i)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            (yrow + (16 * i + r) * ld_y)[lane_y] = from_f32<T>(O[i][r]);
      } else if (active) {
#pragma unroll
        for (int i = 0; i < NB; ++i)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (16 * i + 4 * g + r < nt)
              (yrow + (16 * i + r) * ld_y)[lane_y] = from_f32<T>(O[i][r]);
      }
      // the last chunk has no second one: nobody waits for what follows
      if (at + CH < len) __syncthreads();
    }
    if (active && (COMPOSE || (has_state && ends))) {
#pragma unroll
      for (int i = 0; i < 2 * D; ++i)
        *reinterpret_cast<lm_f32x4*>(to + 16 * i) = S[i];
    }
    return;
  }

  // the convolution's inputs that later tokens look back at
  if (COMPOSE || !has_state || !ends || slice > 0) return;
  const bool own_qk = h % (p.heads / p.groups) == 0;
  const int kv = KP / 8, vv = p.VP / 8, each = 2 * kv + vv;
  const int n = min(sq[3], p.taps - 1);
  for (int i = tid; i < n * each; i += NTH) {
    const int tt = sq[3] - 1 - i / each, j = i % each;
    if (j < 2 * kv && !own_qk) continue;
    const int c = j < kv ? hk * KP + j * 8
                : j < 2 * kv ? p.k_at + hk * KP + (j - kv) * 8
                             : p.v_at + h * p.VP + (j - 2 * kv) * 8;
    copy8(p.ring + ((long)slot * p.taps + (p0 + tt) % p.taps) * p.channels + c,
          p.z + (long)(sq[2] + tt) * p.ld + c);
  }
}

// The state in front of every segment of a portion, in Q's place: a workgroup
// per head, portion and 16 values.
constexpr int CHAIN_COLS = 16;
template <int D, bool DELTA>
__global__ __launch_bounds__(256) void state_chain_kernel(
    const int* __restrict__ seqs, const float* __restrict__ state,
    const float* __restrict__ decay, int n_state, int heads, int VP, int seg,
    const float* __restrict__ P, float* __restrict__ Q) {
  constexpr int KP = D * 32, C4 = KP / 4;
  constexpr int N = CHAIN_COLS * C4, PER = (N + 255) / 256;
  __shared__ __align__(16) float s[CHAIN_COLS][KP];
  const int h = blockIdx.x, v0 = blockIdx.z * CHAIN_COLS;
  const int* sq = seqs + blockIdx.y * 6;
  const int n = segments_of(sq, seg), p0 = sq[4], slot = sq[5];
  int first = 0;  // segments of the portions in front
  for (int b = 0; b < (int)blockIdx.y; ++b)
    first += segments_of(seqs + b * 6, seg);
  const bool has = p0 > 0 && slot >= 0 && slot < n_state;
  const float* st =
      state + (((long)(has ? slot : 0) * heads + h) * VP + v0) * KP;
  for (int i = threadIdx.x; i < N; i += 256)
    *reinterpret_cast<lm_f32x4*>(&s[i / C4][i % C4 * 4]) =
        has ? *reinterpret_cast<const lm_f32x4*>(st + i * 4)
            : lm_f32x4{0.f, 0.f, 0.f, 0.f};
  __syncthreads();
  for (int k = 0; k < n; ++k) {
    const long unit = (long)(first + k) * heads + h;
    float* qc = Q + (unit * VP + v0) * KP;
    const bool more = k + 1 < n;  // else Q and P were not made
    float total = 1.f;
    if (!DELTA && more) {
      const ChunkDecay* d = (const ChunkDecay*)decay +
                            ((long)(sq[0] + k * seg) * heads + h) * 2;
      for (int c = 0; c < 2 * seg; ++c)
        total *= d[(long)(c / 2) * heads * 2 + c % 2].total;
    }
    lm_f32x4 acc[PER];
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int at = threadIdx.x + i * 256;
      if (at >= N) continue;
      const int row = at / C4, c = at % C4 * 4;
      lm_f32x4* q = reinterpret_cast<lm_f32x4*>(qc + at * 4);
      if (more) {
        lm_f32x4 a = *q;
        if (DELTA) {
          const float* pc = P + unit * KP * KP + c;
#pragma unroll 16
          for (int j = 0; j < KP; ++j)
            a += s[row][j] *
                 *reinterpret_cast<const lm_f32x4*>(pc + j * KP);
        } else {
          a += total * *reinterpret_cast<const lm_f32x4*>(&s[row][c]);
        }
        acc[i] = a;
      }
      *q = *reinterpret_cast<const lm_f32x4*>(&s[row][c]);
    }
    if (!more) break;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int at = threadIdx.x + i * 256;
      if (at < N)
        *reinterpret_cast<lm_f32x4*>(&s[at / C4][at % C4 * 4]) = acc[i];
    }
    __syncthreads();
  }
}

// ------------------------------------------------------------------- //
// single tokens: grid (heads, tokens)
// ------------------------------------------------------------------- //
// Eight lanes share a column's keys. D: 32-channel blocks of a key, CL:
// columns of a lane at a time.
template <typename T, int D, int CL, bool DELTA>
__global__ __launch_bounds__(256) void state_step_kernel(StateArgs<T> p) {
  constexpr int KP = D * 32;
  __shared__ __align__(16) float sq[KP];
  __shared__ __align__(16) float sk[KP];
  __shared__ __align__(16) float sv[512];
  __shared__ float part[4];
  const int tid = threadIdx.x, lane = tid & 63;
  const int h = blockIdx.x, t = blockIdx.y;
  const int pos = p.positions[t], slot = p.slots[t];
  const bool has_state = slot >= 0 && slot < p.n_state;
  const bool past = has_state && pos > 0;
  const int per = p.heads / p.groups, hk = h / per;
  const T* z = p.z + (long)t * p.ld;
  const int kg = tid & 7, c0 = tid >> 3;
  float* st = p.state +
              ((long)(has_state ? slot : 0) * p.heads + h) * p.VP * KP +
              kg * 4;
  lm_f32x4 S[CL][D];
  auto load = [&](int base) {
#pragma unroll
    for (int i = 0; i < CL; ++i)
#pragma unroll
      for (int j = 0; j < D; ++j) {
        const int c = base + c0 + 32 * i;
        S[i][j] = lm_f32x4{0.f, 0.f, 0.f, 0.f};
        if (past && c < p.VP)
          S[i][j] = *reinterpret_cast<const lm_f32x4*>(st + (long)c * KP +
                                                       j * 32);
      }
  };
  load(0);
  // convolution
  const int kv = KP / 8, each = 2 * kv + p.VP / 8;
  for (int j = tid; j < each; j += 256) {
    const int c = j < kv ? hk * KP + j * 8
                : j < 2 * kv ? p.k_at + hk * KP + (j - kv) * 8
                             : p.v_at + h * p.VP + (j - 2 * kv) * 8;
    float x[8], w[8], f[8];
    load8<T>(z + c, x);
    load8<T>(p.conv + (long)(p.taps - 1) * p.channels + c, w);
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] = 0.f;
    if (p.conv_b) load8<T>(p.conv_b + c, f);
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] += w[e] * x[e];
    T* ring = p.ring + (long)(has_state ? slot : 0) * p.taps * p.channels + c;
    const int back = has_state ? min(p.taps - 1, pos) : 0;
#pragma unroll
    for (int d = 1; d < MAX_TAPS; ++d) {
      if (d <= back) {
        float r[8];
        load8<T>(ring + (long)((pos - d) % p.taps) * p.channels, r);
        load8<T>(p.conv + (long)(p.taps - 1 - d) * p.channels + c, w);
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] += w[e] * r[e];
      }
    }
    if (has_state && (j >= 2 * kv || h % per == 0))
      copy8(ring + (long)(pos % p.taps) * p.channels, z + c);
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] = silu_f<T>(f[e]);
    store8((j < kv ? sq + j * 8 : j < 2 * kv ? sk + (j - kv) * 8
                                             : sv + (j - 2 * kv) * 8), f);
  }
  float gt, step;
  decay_of(to_f32(z[p.a_at + h]), to_f32(p.a_log[h]), to_f32(p.dt_bias[h]),
           &gt, &step);
  const float decay = expf(gt);
  if (DELTA) step = 1.f / (1.f + expf(-to_f32(z[p.b_at + h])));
  const float skip = DELTA ? 0.f : to_f32(p.skip[h]);
  __syncthreads();
  lm_f32x4 q[D], k[D];
  float nq = 0.f, nk = 0.f;
#pragma unroll
  for (int j = 0; j < D; ++j) {
    q[j] = *reinterpret_cast<const lm_f32x4*>(sq + j * 32 + kg * 4);
    k[j] = *reinterpret_cast<const lm_f32x4*>(sk + j * 32 + kg * 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      nq += q[j][e] * q[j][e];
      nk += k[j][e] * k[j][e];
    }
  }
  if (DELTA) {
    nq = 1.f / (sqrtf(sum8(nq) + 1e-6f) * sqrtf((float)p.dim));
    nk = 1.f / sqrtf(sum8(nk) + 1e-6f);
#pragma unroll
    for (int j = 0; j < D; ++j) {
      q[j] *= nq;
      k[j] *= nk;
    }
  }
  for (int base = 0; base < p.VP; base += 32 * CL) {
    if (base > 0) load(base);
#pragma unroll
    for (int i = 0; i < CL; ++i) {
      const int c = base + c0 + 32 * i;
      const bool live = c < p.VP;  // the same for the eight lanes
      const float v = live ? sv[c] : 0.f;
      float u = step * v;
      if (DELTA) {
        lm_f32x4 a = S[i][0] * k[0];
#pragma unroll
        for (int j = 1; j < D; ++j) a += S[i][j] * k[j];
        u -= step * decay * sum8((a[0] + a[1]) + (a[2] + a[3]));
      }
      lm_f32x4 a = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < D; ++j) {
        S[i][j] = decay * S[i][j] + u * k[j];
        a += S[i][j] * q[j];
        if (live && has_state)
          *reinterpret_cast<lm_f32x4*>(st + (long)c * KP + j * 32) = S[i][j];
      }
      float o = sum8((a[0] + a[1]) + (a[2] + a[3]));
      if (!DELTA) o += skip * v;
      // this column's value has been read by these eight lanes only
      if (live && kg == 0) sv[c] = o;
    }
  }
  __syncthreads();
  if (!DELTA) {
    for (int c = tid; c < p.VP; c += 256)
      p.y[((long)t * p.heads + h) * p.VP + c] = from_f32<T>(sv[c]);
    return;
  }
  float ss = 0.f;
  for (int c = tid; c < p.VP; c += 256) ss += sv[c] * sv[c];
#pragma unroll
  for (int d = 1; d < 64; d <<= 1) ss += __shfl_xor(ss, d, 64);
  if (lane == 0) part[tid >> 6] = ss;
  __syncthreads();
  ss = (part[0] + part[1]) + (part[2] + part[3]);
  const float inv = 1.f / sqrtf(ss / (float)p.vdim + p.eps);
  for (int c = tid; c < p.VP; c += 256)
    p.out[(long)t * p.ld_out + h * p.VP + c] = from_f32<T>(
        sv[c] * inv * to_f32(p.norm[h * p.VP + c]) *
        silu_f<T>(to_f32(z[p.gate_at + h * p.VP + c])));
}

// ------------------------------------------------------------------- //
// norm of the read-outs in parts, gated behind it (DELTA) or in front
// ------------------------------------------------------------------- //
// L threads take a part of a token. VEC 8: parts and heads are multiples of 8.
// KEEP: vectors of a part that a thread keeps between its sum and its norm (0:
// they are read again).
template <typename T, int VEC, int KEEP, bool DELTA>
__global__ __launch_bounds__(256) void state_norm_kernel(StateArgs<T> p,
                                                         int first, int L) {
  __shared__ float part[4];
  const long item = (long)blockIdx.x * (256 / L) + threadIdx.x / L;
  const int lid = threadIdx.x % L;
  const int size = p.heads * p.vdim / p.parts;
  const bool mine = item < (long)(p.n_tok - first) * p.parts;
  const long t = first + (mine ? item / p.parts : 0);
  const int c0 = mine ? (int)(item % p.parts) * size : 0;
  const T* y = p.y + t * p.heads * p.VP;
  const T* gate = p.z + t * p.ld + p.gate_at;
  auto place = [&](int c) { return c / p.vdim * p.VP + c % p.vdim; };
  auto value = [&](int at, float* f) {  // what the norm is of
    if (VEC == 8) load8<T>(y + at, f);
    else f[0] = to_f32(y[at]);
    if (DELTA) return;
    float s[8];
    if (VEC == 8) load8<T>(gate + at, s);
    else s[0] = to_f32(gate[at]);
#pragma unroll
    for (int e = 0; e < VEC; ++e) f[e] *= silu_f<T>(s[e]);
  };
  float ss = 0.f;
  float kept[KEEP ? KEEP : 1][8];
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = (lid + i * L) * VEC;
    if (mine && c < size) {
      value(place(c0 + c), kept[i]);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss += kept[i][e] * kept[i][e];
    }
  }
  if (KEEP == 0 && mine)
    for (int c = lid * VEC; c < size; c += L * VEC) {
      float f[8];
      value(place(c0 + c), f);
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss += f[e] * f[e];
    }
  for (int d = 1; d < min(L, 64); d <<= 1) ss += __shfl_xor(ss, d, 64);
  if (L == 256) {
    if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = ss;
    __syncthreads();
    ss = (part[0] + part[1]) + (part[2] + part[3]);
  }
  if (!mine) return;
  const float inv = 1.f / sqrtf(ss / (float)size + p.eps);
  auto finish = [&](int at, float* f) {
    float w[8];
    if (VEC == 8) load8<T>(p.norm + at, w);
    else w[0] = to_f32(p.norm[at]);
#pragma unroll
    for (int e = 0; e < VEC; ++e) f[e] *= inv * w[e];
    if (DELTA) {
      if (VEC == 8) load8<T>(gate + at, w);
      else w[0] = to_f32(gate[at]);
#pragma unroll
      for (int e = 0; e < VEC; ++e) f[e] *= silu_f<T>(w[e]);
    }
    T* dst = p.out + t * p.ld_out + at;
    if (VEC == 8) store8(dst, f);
    else dst[0] = from_f32<T>(f[0]);
  };
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = (lid + i * L) * VEC;
    if (c < size) finish(place(c0 + c), kept[i]);
  }
  if (KEEP == 0)
    for (int c = lid * VEC; c < size; c += L * VEC) {
      float f[8];
      const int at = place(c0 + c);
      value(at, f);
      finish(at, f);
    }
}

// zeros in the padding of heads whose size is no multiple of 32
template <typename T>
__global__ __launch_bounds__(256) void state_pad_kernel(T* out, long ld_out,
                                                        int heads, int VP,
                                                        int vdim, int n_tok) {
  const int pad = VP - vdim;
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= (long)n_tok * heads * pad) return;
  const long t = i / (heads * pad);
  const int h = (int)(i / pad % heads);
  out[t * ld_out + h * VP + vdim + i % pad] = from_f32<T>(0.f);
}

}  // namespace

// z [T, cols] (row stride free): [q | k | v | gate | a | b], heads padded to
// KP and VP channels; conv [taps, channels]; state [slots, heads, VP, KP]
// float; ring [slots, taps, channels]; tiles [n, 5] of up to `tile` tokens, seqs
// [m, 6] as in rglru; portions are walked in segments of `seg` tiles (0: whole);
// the first n_single tokens are sequences of their own. out [T, heads * VP]
void lm_linear_state(torch::Tensor z, bool delta, long heads, long groups,
                     long dim, long vdim, long parts, double eps,
                     torch::Tensor conv, c10::optional<torch::Tensor> conv_b,
                     torch::Tensor a_log, torch::Tensor dt_bias,
                     c10::optional<torch::Tensor> skip, torch::Tensor norm,
                     torch::Tensor state, torch::Tensor ring,
                     torch::Tensor positions, torch::Tensor slots,
                     torch::Tensor tiles, torch::Tensor seqs, long tile,
                     long seg, long n_single, torch::Tensor out) {
  LM_CHECK_I32(positions);
  LM_CHECK_I32(slots);
  LM_CHECK_I32(tiles);
  LM_CHECK_I32(seqs);
  LM_CHECK_CONTIG(state);
  LM_CHECK_CONTIG(ring);
  const auto type = z.scalar_type();
  const long T = z.size(0);
  TORCH_CHECK(heads >= 1 && groups >= 1 && heads % groups == 0);
  TORCH_CHECK(state.dim() == 4 && state.scalar_type() == at::kFloat &&
              state.size(1) == heads);
  const long VP = state.size(2), KP = state.size(3);
  TORCH_CHECK(VP % 32 == 0 && VP <= 512 && vdim >= 1 && vdim <= VP &&
              dim >= 1 && dim <= KP, "lm_linear_state: head sizes");
  const long C = 2 * groups * KP + heads * VP, SP = (heads + 31) / 32 * 32;
  const long cols = C + heads * VP + (delta ? 2 : 1) * SP;
  lm_check_rows(z, T, cols, type);
  lm_check_rows(out, T, heads * VP, type);
  const long taps = conv.size(0);
  TORCH_CHECK(conv.dim() == 2 && conv.size(1) == C && taps >= 1 &&
              taps <= MAX_TAPS, "lm_linear_state: convolution");
  TORCH_CHECK(ring.dim() == 3 && ring.scalar_type() == type &&
              ring.size(0) == state.size(0) && ring.size(1) == taps &&
              ring.size(2) == C);
  const auto weight = [&](const torch::Tensor& w, long n) {
    LM_CHECK_CONTIG(w);
    TORCH_CHECK(w.numel() == n && w.scalar_type() == type,
                "lm_linear_state: weight");
  };
  weight(conv, taps * C);
  if (conv_b) weight(*conv_b, C);
  weight(a_log, heads);
  weight(dt_bias, heads);
  TORCH_CHECK(delta || skip);
  if (skip) weight(*skip, heads);
  weight(norm, heads * VP);
  TORCH_CHECK(parts >= 1 && heads * vdim % parts == 0 &&
              (!delta || parts == heads));
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 5 && seqs.dim() == 2 &&
              seqs.size(1) == 6);
  const long m = seqs.size(0), nt = tiles.size(0);
  TORCH_CHECK(n_single >= 0 && n_single <= T &&
              positions.numel() >= n_single && slots.numel() >= n_single);
  TORCH_CHECK((m > 0) == (nt > 0) && (m > 0) == (T > n_single));
  TORCH_CHECK(m <= 65535 && n_single <= 65535);
  TORCH_CHECK(tile == TILE, "lm_linear_state: tiles of ", TILE, " tokens");
  TORCH_CHECK(seg >= 0 && nt >= m);
  // every portion's last segment may be short
  const long n_seg = seg && m ? (nt - m) / seg + m : 0;
  TORCH_CHECK(n_seg <= 65535);
  if (T == 0) return;
  const auto opt = z.options();
  auto u = torch::empty({m > 0 ? T - n_single + CH : 0, C}, opt);
  auto y = torch::empty({T, heads * VP}, opt);
  auto decay = torch::empty({nt * heads * 2 * DECAY}, state.options());
  torch::Tensor P, Q;
  if (n_seg) {
    if (delta) P = torch::empty({n_seg, heads, KP, KP}, state.options());
    Q = torch::empty({n_seg, heads, VP, KP}, state.options());
  }
  hipStream_t st = cmls::current_stream();
#define LM_ST_(D, CL, DELTA)                                                \
  hipLaunchKernelGGL((state_step_kernel<scalar_t, D, CL, DELTA>),           \
                     dim3(heads, n_single), dim3(256), 0, st, a)
#define LM_ST(D, CL)                                                        \
  do { if (delta) LM_ST_(D, CL, true); else LM_ST_(D, CL, false); } while (0)
#define LM_ST_D(D)                                                          \
  do {                                                                      \
    if (VP <= 64) LM_ST(D, 2);                                         \
    else LM_ST(D, 4);                                                       \
  } while (0)
#define LM_SC_(TAPS, DELTA)                                                 \
  hipLaunchKernelGGL((state_conv_kernel<scalar_t, TAPS, DELTA>), cg,        \
                     dim3(256), 0, st, a, n_conv)
#define LM_SC(TAPS)                                                         \
  do { if (delta) LM_SC_(TAPS, true); else LM_SC_(TAPS, false); } while (0)
#define LM_CK__(D, DELTA, COMPOSE, COLS, ROWS)                              \
  do {                                                                      \
    const int bytes = (4 * CH * (KP + 4) +                                  \
                       (DELTA ? 4 : 2) * CH * (CH + 4) + 2 * DECAY) * 4;    \
    auto* fn = &state_chunk_kernel<scalar_t, D, DELTA, COMPOSE>;            \
    HIP_CHECK(hipFuncSetAttribute(                                          \
        reinterpret_cast<const void*>(fn),                                  \
        hipFuncAttributeMaxDynamicSharedMemorySize, bytes));                \
    hipLaunchKernelGGL(fn, dim3(heads * ((COLS + NW * 16 - 1) / (NW * 16)), \
                                ROWS), dim3(2 * NTH), bytes, st, a);        \
  } while (0)
#define LM_CK_(D, DELTA)                                                    \
  do {                                                                      \
    if (seg) {                                                              \
      LM_CK__(D, DELTA, true, (DELTA ? KP : 0) + VP, n_seg);                \
      hipLaunchKernelGGL((state_chain_kernel<D, DELTA>),                    \
                         dim3(heads, m, VP / CHAIN_COLS), dim3(256), 0, st, \
                         a.seqs, a.state, a.decay, a.n_state, a.heads,      \
                         (int)VP, (int)seg, a.P, a.Q);                      \
    }                                                                       \
    LM_CK__(D, DELTA, false, VP, seg ? n_seg : m);                          \
  } while (0)
#define LM_CK(D)                                                            \
  do { if (delta) LM_CK_(D, true); else LM_CK_(D, false); } while (0)
#define LM_SN(VEC, KEEP, DELTA)                                             \
  hipLaunchKernelGGL((state_norm_kernel<scalar_t, VEC, KEEP, DELTA>), grid, \
                     dim3(256), 0, st, a, (int)first, L)
#define LM_SN_K(VEC, DELTA)                                                 \
  do {                                                                      \
    if (n_vec <= L) LM_SN(VEC, 1, DELTA);                                   \
    else if (keep) LM_SN(VEC, 4, DELTA);                                    \
    else LM_SN(VEC, 0, DELTA);                                              \
  } while (0)
  LM_DISPATCH(z, "lm_linear_state", [&] {
    const auto ptr = [](const torch::Tensor& w) {
      return (const scalar_t*)w.data_ptr();
    };
    StateArgs<scalar_t> a{};
    a.z = ptr(z);
    a.ld = z.stride(0);
    a.k_at = (int)(groups * KP);
    a.v_at = 2 * a.k_at;
    a.channels = a.gate_at = (int)C;
    a.a_at = (int)(C + heads * VP);
    a.b_at = a.a_at + (int)SP;
    a.conv = ptr(conv);
    a.conv_b = conv_b ? ptr(*conv_b) : nullptr;
    a.a_log = ptr(a_log);
    a.dt_bias = ptr(dt_bias);
    a.skip = skip ? ptr(*skip) : nullptr;
    a.norm = ptr(norm);
    a.state = state.data_ptr<float>();
    a.ring = (scalar_t*)ring.data_ptr();
    a.u = (scalar_t*)u.data_ptr();
    a.decay = decay.data_ptr<float>();
    a.y = (scalar_t*)y.data_ptr();
    a.out = (scalar_t*)out.data_ptr();
    a.ld_out = out.stride(0);
    a.positions = positions.data_ptr<int>();
    a.slots = slots.data_ptr<int>();
    a.tiles = tiles.data_ptr<int>();
    a.seqs = seqs.data_ptr<int>();
    a.n_single = (int)n_single;
    a.n_seq = (int)m;
    a.n_state = (int)state.size(0);
    a.n_tok = (int)T;
    a.heads = (int)heads;
    a.groups = (int)groups;
    a.KP = (int)KP;
    a.VP = (int)VP;
    a.dim = (int)dim;
    a.vdim = (int)vdim;
    a.taps = (int)taps;
    a.parts = (int)parts;
    a.eps = (float)eps;
    a.seg = n_seg ? (int)seg : 0;
    a.n_seg = (int)n_seg;
    if (n_seg) {
      a.P = delta ? P.data_ptr<float>() : nullptr;
      a.Q = Q.data_ptr<float>();
    }

    if (n_single > 0) {
      switch (KP) {
        case 32: LM_ST_D(1); break;
        case 64: LM_ST_D(2); break;
        case 96: LM_ST_D(3); break;
        case 128: LM_ST_D(4); break;
        case 256: LM_ST_D(8); break;
        default: TORCH_CHECK(false, "lm_linear_state: keys of ", KP);
      }
    }
    if (m > 0) {
      const int n_conv = (int)(C / 8 + 31) / 32;
      const dim3 cg(nt, n_conv + (heads + 3) / 4);
      if (taps <= 2) LM_SC(2);
      else if (taps <= 4) LM_SC(4);
      else LM_SC(MAX_TAPS);
      switch (KP) {
        case 32: LM_CK(1); break;
        case 64: LM_CK(2); break;
        case 96: LM_CK(3); break;
        case 128: LM_CK(4); break;
        case 256: LM_CK(8); break;
        default: TORCH_CHECK(false, "lm_linear_state: keys of ", KP);
      }
    }
    // the step kernel has finished single tokens of the delta rule
    const long first = delta ? n_single : 0;
    const long size = heads * vdim / parts;
    const bool vec = vdim % 8 == 0 && size % 8 == 0;
    if (VP > vdim && first < T) {
      const long n = (T - first) * heads * (VP - vdim);
      hipLaunchKernelGGL((state_pad_kernel<scalar_t>),
                         dim3((n + 255) / 256), dim3(256), 0, st,
                         a.out + first * a.ld_out, a.ld_out, (int)heads,
                         (int)VP, (int)vdim, (int)(T - first));
    }
    if (first < T) {
      // up to four vectors of a thread of a wave, else a workgroup per part
      const long n_vec = (size + (vec ? 7 : 0)) / (vec ? 8 : 1);
      int L = 4;
      while (L < 64 && L < n_vec) L *= 2;
      if (n_vec > 256) L = 256;
      const bool keep = n_vec <= 4L * L;
      const long items = (T - first) * parts;
      const dim3 grid((items + 256 / L - 1) / (256 / L));
      if (vec && delta) LM_SN_K(8, true);
      else if (vec) LM_SN_K(8, false);
      else if (delta) LM_SN_K(1, true);
      else LM_SN_K(1, false);
    }
  });
#undef LM_ST_D
#undef LM_ST
#undef LM_ST_
#undef LM_SC
#undef LM_SC_
#undef LM_CK
#undef LM_CK_
#undef LM_CK__
#undef LM_SN
#undef LM_SN_K
  LM_LAUNCHED();
}
