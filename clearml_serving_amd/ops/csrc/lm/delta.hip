// Generalised delta rule: per head a state S [key][value], float, and per token
//
//   w = exp(-e^(-1/2) sigmoid(W2 tanh(z) + w0))     decay of a key channel
//   a = sigmoid(za + ba)                            removal rate
//   u = k / |k|                                     unit key
//   S <- diag(w) S - (a u) (u^T S) + k v^T,   o = S^T r
//   out = o / rms(o) * norm * sigmoid(zg)
//
// r, k, v, za, zg and z (the low-rank input of the decay) are projections of the
// same input; all else is float. The columns of S do not depend on each other,
// so a workgroup keeps the whole state of one (sequence, head) in registers and
// walks the sequence's tokens: a wave takes a range of columns, eight lanes
// share a column's rows, sums over them are DPP adds. k v^T is taken as
// u (|k| v)^T, so u is read once for both. The tokens' vectors are
// made in tiles of 16 through LDS -- the low-rank product by MFMA in 32-bit,
// next tile's projections in flight meanwhile -- and the outputs are normed and
// gated from there. Single tokens are portions of one: same kernel.
//
// Few long portions would leave most CUs idle, so these are cut into chunks. A
// token's step is S <- A S + k v^T; a chunk's is S <- P S + Q. The same walk
// makes P, from the identity without values, and Q, from zero; a chain over the
// chunks gives the state in front of each (delta_chain_kernel), and the chunks
// are walked again from there, now with outputs.
//
// State in memory: [slot][head][value][key]. Slots are never cleared: position
// 0 starts from zero.
#include "lm_attn.h"

namespace {

constexpr int TT = 16;  // tokens per tile

// sum over the eight lanes that share lane >> 3
__device__ __forceinline__ float sum8(float v) {
  v += __int_as_float(__builtin_amdgcn_update_dpp(
      0, __float_as_int(v), 0xB1, 0xf, 0xf, true));  // quad_perm 1 0 3 2
  v += __int_as_float(__builtin_amdgcn_update_dpp(
      0, __float_as_int(v), 0x4E, 0xf, 0xf, true));  // quad_perm 2 3 0 1
  v += __int_as_float(__builtin_amdgcn_update_dpp(
      0, __float_as_int(v), 0x141, 0xf, 0xf, true));  // row_half_mirror
  return v;
}

template <typename T> struct Four;
template <> struct Four<bf16> { uint2 u; };
template <> struct Four<float> { lm_f32x4 u; };
template <typename T> __device__ __forceinline__ Four<T> load4(const T* p) {
  Four<T> f;
  f.u = *reinterpret_cast<const decltype(f.u)*>(p);
  return f;
}
__device__ __forceinline__ lm_f32x4 floats(const Four<bf16>& v) {
  union { uint2 u; bf16 b[4]; } c;
  c.u = v.u;
  return lm_f32x4{to_f32(c.b[0]), to_f32(c.b[1]), to_f32(c.b[2]),
                  to_f32(c.b[3])};
}
__device__ __forceinline__ lm_f32x4 floats(const Four<float>& v) {
  return v.u;
}

template <typename T>
struct DeltaArgs {
  const T* z;  // projections, rows of ld
  long ld;
  int r, k, v, g, a, w1;          // columns of the parts
  const T *w2, *w0, *ab, *norm;   // [heads * DP, RP], [heads * DP] each
  T* out;                         // rows of ld_out, head h at h * DP
  long ld_out;
  float* state;                   // [slots, heads, DP, DP]
  const int *positions, *slots, *seqs;
  int n_single, n_seq, n_state, heads, dim, RP;
  float eps, out_scale;
  // chunks of `chunk` tiles of `tile` tokens; 0: whole portions
  int n_chunks, tile, chunk;      // n_chunks: bound on all portions' chunks
  float *P, *Q;                   // [n_chunks, heads, DP, DP]
};

__device__ __forceinline__ int chunks_of(const int* portion, int chunk) {
  return (portion[1] + chunk - 1) / chunk;
}

// D: 32-channel blocks of a head, NW: waves. COMPOSE: a chunk's P (grid z 1)
// or Q (grid z 0) instead of outputs.
template <typename T, int D, int NW, bool COMPOSE>
__global__ __launch_bounds__(NW * 64, NW == 4 && D <= 2 ? 2 : 1)
void delta_rule_kernel(DeltaArgs<T> p) {
  constexpr int DP = D * 32, NTH = NW * 64;
  constexpr int CL = DP / (8 * NW);                    // columns of a lane
  constexpr int CT = (DP / 16 + NW - 1) / NW;          // channel tiles of a wave
  constexpr int OC = DP / 4;                           // threads per output row
  constexpr int ON = (TT * OC + NTH - 1) / NTH;
  static_assert(CL * 8 * NW == DP && CL >= 1, "columns");
  extern __shared__ __align__(16) float sm[];
  float* su = sm;                // [TT][DP] each
  float* sb = su + TT * DP;
  float* sw = sb + TT * DP;
  float* sr = sw + TT * DP;
  float* sv = sr + TT * DP;      // values times |k|, then outputs
  float* ssq = sv + TT * DP;     // [NW][TT]
  const int tid = threadIdx.x, lane = tid & 63, wave = uniform_wave();
  const int r16 = lane & 15, g = lane >> 4;
  const int kg = lane & 7, cg = lane >> 3;
  const int h = blockIdx.x;

  int t0, len, p0, slot;
  const float* start = nullptr;  // state in front of a chunk
  float* made = nullptr;         // where P or Q goes
  bool ends = true;              // the portion ends here
  const int n_work = p.chunk ? p.n_chunks : p.n_seq;
  if (p.chunk && (int)blockIdx.y < n_work) {
    int c = blockIdx.y, s = 0;  // chunk c of portion s
    while (s < p.n_seq && c >= chunks_of(p.seqs + s * 6, p.chunk))
      c -= chunks_of(p.seqs + s++ * 6, p.chunk);
    if (s == p.n_seq) return;
    const int* sd = p.seqs + s * 6;
    ends = (c + 1) * p.chunk >= sd[1];
    if (COMPOSE && ends) return;  // nothing follows
    const int skip = c * p.chunk * p.tile;
    t0 = sd[2] + skip;
    len = min(p.chunk * p.tile, sd[3] - skip);
    p0 = sd[4] + skip;
    slot = sd[5];
    const long at = ((long)blockIdx.y * p.heads + h) * DP * DP;
    start = p.Q + at;
    made = (blockIdx.z ? p.P : p.Q) + at;
  } else if ((int)blockIdx.y < n_work) {
    // long sequences first: they are the last of the list
    const int* sd = p.seqs + (p.n_seq - 1 - (int)blockIdx.y) * 6;
    t0 = sd[2], len = sd[3], p0 = sd[4], slot = sd[5];
  } else {
    t0 = blockIdx.y - n_work;
    len = 1;
    p0 = p.positions[t0];
    slot = p.slots[t0];
  }
  const bool has_state = slot >= 0 && slot < p.n_state;
  float* st = p.state + ((long)(has_state ? slot : 0) * p.heads + h) * DP * DP;

  // lane's part of the state: columns c0 + i, rows 32 j + 4 kg + e
  const int c0 = wave * (DP / NW) + cg * CL;
  lm_f32x4 S[CL][D];
#pragma unroll
  for (int i = 0; i < CL; ++i)
#pragma unroll
    for (int j = 0; j < D; ++j)
      S[i][j] = lm_f32x4{0.f, 0.f, 0.f, 0.f};
  if (COMPOSE) {
    if (blockIdx.z) {
#pragma unroll
      for (int i = 0; i < CL; ++i)
#pragma unroll
        for (int j = 0; j < D; ++j)
#pragma unroll
          for (int e = 0; e < 4; ++e)
            S[i][j][e] = j * 32 + kg * 4 + e == c0 + i ? 1.f : 0.f;
    }
  } else if (start || (p0 > 0 && has_state)) {
    const float* from = start ? start : st;
#pragma unroll
    for (int i = 0; i < CL; ++i)
#pragma unroll
      for (int j = 0; j < D; ++j)
        S[i][j] = *reinterpret_cast<const lm_f32x4*>(
            from + (c0 + i) * DP + j * 32 + kg * 4);
  }

  // a lane prepares channels ch[c] + [0, 4) of token r16 of a tile
  bool live[CT];
  int ch[CT];
  lm_f32x4 w0[CT], ab[CT];
#pragma unroll
  for (int c = 0; c < CT; ++c) {
    const int tile = wave + c * NW;
    live[c] = tile < DP / 16;  // uniform in the wave
    ch[c] = (live[c] ? tile : 0) * 16 + 4 * g;
    w0[c] = floats(load4(p.w0 + h * DP + ch[c]));
    ab[c] = floats(load4(p.ab + h * DP + ch[c]));
  }
  Four<T> fr[CT], fk[CT], fv[CT], fa[CT];
  auto load = [&](int at) {
    const T* row = p.z + (long)(t0 + min(at + r16, len - 1)) * p.ld + h * DP;
#pragma unroll
    for (int c = 0; c < CT; ++c) {
      fr[c] = load4(row + p.r + ch[c]);
      fk[c] = load4(row + p.k + ch[c]);
      fv[c] = load4(row + p.v + ch[c]);
      fa[c] = load4(row + p.a + ch[c]);
    }
  };
  load(0);
  const T* w2 = p.w2 + (long)h * DP * p.RP;

  for (int at = 0; at < len; at += TT) {
    const int nt = min(TT, len - at);
    // low-rank part of the decay: C row = channel, column = token
    lm_f32x4 zw[CT];
#pragma unroll
    for (int c = 0; c < CT; ++c) zw[c] = w0[c];
    {
      const T* zr = p.z + (long)(t0 + min(at + r16, len - 1)) * p.ld + p.w1 +
                    g * 8;
      for (int k = 0; k < p.RP; k += 32) {
        Frag<float> tf;
        load8<T>(zr + k, tf.v);
#pragma unroll
        for (int e = 0; e < 8; ++e) tf.v[e] = cap_tanh<T>(tf.v[e]);
#pragma unroll
        for (int c = 0; c < CT; ++c) {
          if (live[c]) {
            Frag<float> wf;
            load8<T>(w2 + (long)(ch[c] - 4 * g + r16) * p.RP + k + g * 8,
                     wf.v);
            zw[c] = mma32(wf, tf, zw[c]);
          }
        }
      }
    }
    float sq = 0.f;
#pragma unroll
    for (int c = 0; c < CT; ++c) {
      if (live[c]) {
        const lm_f32x4 k = floats(fk[c]);
        sq += k[0] * k[0] + k[1] * k[1] + k[2] * k[2] + k[3] * k[3];
      }
    }
    sq += __shfl_xor(sq, 16, 64);
    sq += __shfl_xor(sq, 32, 64);
    if (g == 0) ssq[wave * TT + r16] = sq;
    __syncthreads();  // also: the previous tile's outputs have been read
    sq = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) sq += ssq[w * TT + r16];
    const float size = sqrtf(sq + 1e-6f), inv = 1.f / size;
#pragma unroll
    for (int c = 0; c < CT; ++c) {
      if (live[c]) {
        const lm_f32x4 k = floats(fk[c]), za = floats(fa[c]);
        lm_f32x4 u, b, w;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          u[e] = k[e] * inv;
          b[e] = sigmoid_f(za[e] + ab[c][e]) * u[e];
          // e^(-1/2)
          w[e] = exp_f(-0.60653065971263342f * sigmoid_f(zw[c][e]));
        }
        const int o = r16 * DP + ch[c];
        *reinterpret_cast<lm_f32x4*>(su + o) = u;
        *reinterpret_cast<lm_f32x4*>(sb + o) = b;
        *reinterpret_cast<lm_f32x4*>(sw + o) = w;
        if (!COMPOSE) *reinterpret_cast<lm_f32x4*>(sr + o) = floats(fr[c]);
        *reinterpret_cast<lm_f32x4*>(sv + o) =
            COMPOSE && blockIdx.z ? lm_f32x4{0.f, 0.f, 0.f, 0.f}
                                  : size * floats(fv[c]);
      }
    }
    __syncthreads();
    if (at + TT < len) load(at + TT);
    Four<T> fg[ON];
#pragma unroll
    for (int i = 0; i < (COMPOSE ? 0 : ON); ++i) {
      const int q = tid + i * NTH, tt = min(q / OC, nt - 1);
      fg[i] = load4(p.z + (long)(t0 + at + tt) * p.ld + p.g + h * DP +
                    q % OC * 4);
    }

    for (int t = 0; t < nt; ++t) {
      const int o = t * DP + kg * 4;
      lm_f32x4 u[D], b[D], w[D], r[D];
#pragma unroll
      for (int j = 0; j < D; ++j) {
        u[j] = *reinterpret_cast<const lm_f32x4*>(su + o + j * 32);
        b[j] = *reinterpret_cast<const lm_f32x4*>(sb + o + j * 32);
        w[j] = *reinterpret_cast<const lm_f32x4*>(sw + o + j * 32);
        if (!COMPOSE) r[j] = *reinterpret_cast<const lm_f32x4*>(sr + o + j * 32);
      }
      float y[CL];
#pragma unroll
      for (int i = 0; i < CL; ++i) {
        const float v = sv[t * DP + c0 + i];
        lm_f32x4 a4 = u[0] * S[i][0];
#pragma unroll
        for (int j = 1; j < D; ++j) a4 += u[j] * S[i][j];
        const float x = sum8((a4[0] + a4[1]) + (a4[2] + a4[3]));
        lm_f32x4 y4 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < D; ++j) {
          S[i][j] = w[j] * S[i][j] + (u[j] * v - b[j] * x);
          if (!COMPOSE) y4 += r[j] * S[i][j];
        }
        y[i] = (y4[0] + y4[1]) + (y4[2] + y4[3]);
      }
#pragma unroll
      for (int i = 0; i < (COMPOSE ? 0 : CL); ++i) {
        y[i] = sum8(y[i]);
        // this column's value has been read by these eight lanes only
        if (kg == 0) sv[t * DP + c0 + i] = y[i];
      }
    }
    __syncthreads();

    // norm over the head, weight, gate
#pragma unroll
    for (int i = 0; i < (COMPOSE ? 0 : ON); ++i) {
      const int q = tid + i * NTH, tt = q / OC, c = q % OC * 4;
      lm_f32x4 o = {0.f, 0.f, 0.f, 0.f};
      if (tt < nt) o = *reinterpret_cast<const lm_f32x4*>(sv + tt * DP + c);
      float ss = o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3];
      if ((OC & (OC - 1)) == 0) {  // a row's threads lie in one wave
#pragma unroll
        for (int e = 1; e < OC; e <<= 1) ss += __shfl_xor(ss, e, 64);
      } else if (tt < nt) {
        ss = 0.f;
        for (int e = 0; e < DP; e += 4) {
          const lm_f32x4 f =
              *reinterpret_cast<const lm_f32x4*>(sv + tt * DP + e);
          ss += f[0] * f[0] + f[1] * f[1] + f[2] * f[2] + f[3] * f[3];
        }
      }
      if (tt >= nt) continue;
      const float iv = p.out_scale / sqrtf(ss / (float)p.dim + p.eps);
      const lm_f32x4 nw = floats(load4(p.norm + h * DP + c));
      const lm_f32x4 zg = floats(fg[i]);
      float f[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) f[e] = o[e] * iv * nw[e] * sigmoid_f(zg[e]);
      store4(p.out + (long)(t0 + at + tt) * p.ld_out + h * DP + c, f);
    }
  }

  if (!COMPOSE && !(has_state && ends)) return;
  float* to = COMPOSE ? made : st;
#pragma unroll
  for (int i = 0; i < CL; ++i)
#pragma unroll
    for (int j = 0; j < D; ++j)
      *reinterpret_cast<lm_f32x4*>(to + (c0 + i) * DP + j * 32 + kg * 4) =
          S[i][j];
}

// The state in front of every chunk of a portion, in Q's place: one workgroup
// per head, portion and 16 columns of the state.
constexpr int CHAIN_COLS = 16;
template <int D>
__global__ __launch_bounds__(256) void delta_chain_kernel(
    const int* __restrict__ seqs, const float* __restrict__ state,
    int n_state, int heads, int chunk, const float* __restrict__ P,
    float* __restrict__ Q) {
  constexpr int DP = D * 32, C4 = DP / 4;
  constexpr int N = CHAIN_COLS * C4, PER = (N + 255) / 256;
  __shared__ __align__(16) float s[CHAIN_COLS][DP];
  const int h = blockIdx.x, v0 = blockIdx.z * CHAIN_COLS;
  const int* sd = seqs + blockIdx.y * 6;
  const int n = chunks_of(sd, chunk), p0 = sd[4], slot = sd[5];
  int first = 0;  // chunks of the portions in front
  for (int b = 0; b < (int)blockIdx.y; ++b)
    first += chunks_of(seqs + b * 6, chunk);
  const bool has = p0 > 0 && slot >= 0 && slot < n_state;
  const float* st =
      state + (((long)(has ? slot : 0) * heads + h) * DP + v0) * DP;
  for (int g = threadIdx.x; g < N; g += 256)
    *reinterpret_cast<lm_f32x4*>(&s[g / C4][g % C4 * 4]) =
        has ? *reinterpret_cast<const lm_f32x4*>(st + g * 4)
            : lm_f32x4{0.f, 0.f, 0.f, 0.f};
  __syncthreads();
  for (int k = 0; k < n; ++k) {
    const long at = ((long)(first + k) * heads + h) * DP * DP;
    const float* pc = P + at;
    float* qc = Q + at + v0 * DP;
    const bool more = k + 1 < n;  // else Q and P were not made
    lm_f32x4 acc[PER];
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int g = threadIdx.x + i * 256;
      if (g >= N) continue;
      const int row = g / C4, c = g % C4 * 4;
      lm_f32x4* q = reinterpret_cast<lm_f32x4*>(qc + g * 4);
      if (more) {
        lm_f32x4 a = *q;
#pragma unroll 16
        for (int j = 0; j < DP; ++j)
          a += s[row][j] * *reinterpret_cast<const lm_f32x4*>(pc + j * DP + c);
        acc[i] = a;
      }
      *q = *reinterpret_cast<const lm_f32x4*>(&s[row][c]);
    }
    if (!more) break;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int g = threadIdx.x + i * 256;
      if (g < N)
        *reinterpret_cast<lm_f32x4*>(&s[g / C4][g % C4 * 4]) = acc[i];
    }
    __syncthreads();
  }
}

}  // namespace

// z [T, cols]: columns at[] = r, k, v, g, a (heads * DP each), w1 (RP); w2
// [heads * DP, RP]; seqs [m, 6] as in rglru; the first n_single tokens are
// sequences of their own. out [T, heads * DP], row stride free. Portions are
// cut into chunks of `chunk` tiles of `tile` tokens, 0: not at all; n_tiles:
// tiles of all portions.
void lm_delta_rule(torch::Tensor z, std::vector<long> at, torch::Tensor w2,
                   torch::Tensor w0, torch::Tensor ab, torch::Tensor norm,
                   torch::Tensor state, torch::Tensor positions,
                   torch::Tensor slots, torch::Tensor seqs, torch::Tensor out,
                   long n_single, long dim, double eps, double out_scale,
                   long n_tiles, long tile, long chunk) {
  LM_CHECK_I32(positions);
  LM_CHECK_I32(slots);
  LM_CHECK_I32(seqs);
  const auto type = z.scalar_type();
  TORCH_CHECK(state.is_cuda() && state.is_contiguous() && state.dim() == 4 &&
              state.scalar_type() == at::kFloat &&
              state.size(2) == state.size(3));
  const int heads = state.size(1), DP = state.size(2), T = z.size(0);
  const long HD = (long)heads * DP, RP = w2.size(1);
  TORCH_CHECK(z.is_cuda() && z.dim() == 2 && z.stride(1) == 1 &&
              z.stride(0) % 8 == 0 && z.storage_offset() % 8 == 0);
  TORCH_CHECK(at.size() == 6, "lm_delta_rule: six parts");
  for (int i = 0; i < 6; ++i)
    TORCH_CHECK(at[i] >= 0 && at[i] % 8 == 0 &&
                at[i] + (i < 5 ? HD : RP) <= z.size(1));
  TORCH_CHECK(RP % 32 == 0 && w2.dim() == 2 && w2.size(0) == HD);
  for (const auto* w : {&w2, &w0, &ab, &norm})
    TORCH_CHECK(w->is_cuda() && w->is_contiguous() &&
                w->scalar_type() == type);
  TORCH_CHECK(w0.numel() == HD && ab.numel() == HD && norm.numel() == HD);
  TORCH_CHECK(seqs.dim() == 2 && seqs.size(1) == 6);
  TORCH_CHECK(n_single >= 0 && n_single <= T && positions.numel() >= n_single &&
              slots.numel() >= n_single);
  TORCH_CHECK(out.dim() == 2 && out.size(0) == T && out.size(1) == HD &&
              out.stride(1) == 1 && out.stride(0) % 8 == 0 &&
              out.storage_offset() % 8 == 0 && out.scalar_type() == type);
  TORCH_CHECK(dim >= 1 && dim <= DP);
  const int m = seqs.size(0);
  if (m + n_single == 0) return;
  TORCH_CHECK(chunk >= 0 && tile >= 1 && n_tiles >= m);
  if (m == 0) chunk = 0;
  // every portion's last chunk may be short
  const long n_chunks = chunk ? (n_tiles - m) / chunk + m : 0;
  const long work = (chunk ? n_chunks : m) + n_single;
  TORCH_CHECK(work <= 65535);
  torch::Tensor P, Q;
  if (chunk) {
    P = torch::empty({n_chunks, heads, DP, DP}, state.options());
    Q = torch::empty_like(P);
  }
  hipStream_t stream = cmls::current_stream();
#define LM_DR_(D, NW, COMPOSE, GRID)                                         \
  do {                                                                       \
    const int bytes = (5 * TT * DP + NW * TT) * 4;                           \
    auto* fn = &delta_rule_kernel<scalar_t, D, NW, COMPOSE>;                 \
    HIP_CHECK(hipFuncSetAttribute(                                           \
        reinterpret_cast<const void*>(fn),                                   \
        hipFuncAttributeMaxDynamicSharedMemorySize, bytes));                 \
    hipLaunchKernelGGL(fn, GRID, dim3(NW * 64), bytes, stream, a);           \
  } while (0)
#define LM_DR(D, NW)                                                         \
  do {                                                                       \
    if (chunk) {                                                             \
      LM_DR_(D, NW, true, dim3(heads, n_chunks, 2));                         \
      hipLaunchKernelGGL((delta_chain_kernel<D>),                            \
                         dim3(heads, m, DP / CHAIN_COLS), dim3(256), 0,      \
                         stream, a.seqs, state.data_ptr<float>(), a.n_state, \
                         heads, (int)chunk, a.P, a.Q);                       \
    }                                                                        \
    LM_DR_(D, NW, false, dim3(heads, work));                                 \
  } while (0)
  LM_DISPATCH(z, "lm_delta_rule", [&] {
    DeltaArgs<scalar_t> a{};
    a.z = (const scalar_t*)z.data_ptr();
    a.ld = z.stride(0);
    a.r = (int)at[0];
    a.k = (int)at[1];
    a.v = (int)at[2];
    a.g = (int)at[3];
    a.a = (int)at[4];
    a.w1 = (int)at[5];
    a.w2 = (const scalar_t*)w2.data_ptr();
    a.w0 = (const scalar_t*)w0.data_ptr();
    a.ab = (const scalar_t*)ab.data_ptr();
    a.norm = (const scalar_t*)norm.data_ptr();
    a.out = (scalar_t*)out.data_ptr();
    a.ld_out = out.stride(0);
    a.state = state.data_ptr<float>();
    a.positions = positions.data_ptr<int>();
    a.slots = slots.data_ptr<int>();
    a.seqs = seqs.data_ptr<int>();
    a.n_single = (int)n_single;
    a.n_seq = m;
    a.n_state = (int)state.size(0);
    a.heads = heads;
    a.dim = (int)dim;
    a.RP = (int)RP;
    a.eps = (float)eps;
    a.out_scale = (float)out_scale;
    a.n_chunks = (int)n_chunks;
    a.tile = (int)tile;
    a.chunk = (int)chunk;
    if (chunk) {
      a.P = P.data_ptr<float>();
      a.Q = Q.data_ptr<float>();
    }
    switch (DP) {
      case 32: LM_DR(1, 4); break;
      case 64: LM_DR(2, 4); break;
      case 96: LM_DR(3, 4); break;
      case 128: LM_DR(4, 4); break;
      case 192: LM_DR(6, 8); break;
      case 256: LM_DR(8, 8); break;
      default: TORCH_CHECK(false, "lm_delta_rule: head of ", DP, " channels");
    }
  });
#undef LM_DR
#undef LM_DR_
  LM_LAUNCHED();
}
