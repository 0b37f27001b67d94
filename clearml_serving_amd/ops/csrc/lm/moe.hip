// Mixture of experts on a flat token batch: routing, grouping by expert and
// the grouped products.
//
// Every token takes `top` experts. Its T * top slots are put in expert order
// (pos: slot -> row, tok: row -> token); a tile list cuts each expert's rows
// into pieces of at most `rows` rows. A grouped product runs one workgroup per
// (tile, column range) and takes its row count from the list, so nothing is
// read back to the host. Shared experts, which every token takes, are slots
// behind the `top` chosen ones; identity experts, whose output is the input,
// have no rows (pos -1). The list's length lies in device memory: a launch
// covers the most tiles there can be and the surplus workgroups leave at once.
// A row's result does not depend on where its expert's rows end up.
#include "lm_common.h"

namespace {

constexpr int RT = 16;  // tokens per routing workgroup
constexpr int MAX_TOP = 64;

// Rows and tiles in front of each expert, by a whole workgroup (>= 64
// threads). off: E row offsets; with `tiles` also the tile list.
__device__ void scan_experts(const int* tot, int* off, int E, int rows,
                             int* tiles, int* n_tiles) {
  __shared__ int t_off[1024];
  if (threadIdx.x < 64) {
    const int lane = threadIdx.x;
    int row_base = 0, tile_base = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int e = e0 + lane;
      const int c = e < E ? tot[e] : 0;
      const int nt = (c + rows - 1) / rows;
      int rs = c, ts = nt;
#pragma unroll
      for (int d = 1; d < 64; d <<= 1) {
        const int r = __shfl_up(rs, d, 64), t = __shfl_up(ts, d, 64);
        if (lane >= d) { rs += r; ts += t; }
      }
      if (e < E) {
        off[e] = row_base + rs - c;
        t_off[e] = tile_base + ts - nt;
      }
      row_base += __shfl(rs, 63, 64);
      tile_base += __shfl(ts, 63, 64);
    }
    if (tiles && lane == 0) n_tiles[0] = tile_base;
  }
  __syncthreads();
  if (!tiles) return;
  for (int e = threadIdx.x; e < E; e += blockDim.x) {
    const int c = tot[e];
    for (int j = 0, r = 0; r < c; ++j, r += rows) {
      int* d = tiles + (t_off[e] + j) * 3;
      d[0] = e;
      d[1] = off[e] + r;
      d[2] = min(rows, c - r);
    }
  }
}

// partial logits of 16 tokens and NE * 16 experts over [k_lo, k_hi); a result
// row is an expert, a column (lane & 15) a token
template <typename T, int NE>
__device__ __forceinline__ void router_tiles(const T* hr, const T* router,
                                             int e0, int E, int K, int k_lo,
                                             int k_hi, float* part) {
  const int lane = threadIdx.x & 63, r16 = lane & 15, g = lane >> 4;
  lm_f32x4 acc[NE];
  const T* wr[NE];
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    acc[i] = lm_f32x4{0.f, 0.f, 0.f, 0.f};
    wr[i] = router + (long)min(e0 + i * 16 + r16, E - 1) * K;
  }
#pragma unroll 4
  for (int k = k_lo; k < k_hi; k += 32) {
    const Frag<T> hf = load_frag(hr + k);
#pragma unroll
    for (int i = 0; i < NE; ++i)
      acc[i] = mma32(load_frag(wr[i] + k), hf, acc[i]);
  }
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const float f[4] = {acc[i][0], acc[i][1], acc[i][2], acc[i][3]};
    store4(part + i * 16 + 4 * g, f);
  }
}

// How the chosen experts are found and weighed.
// over_all: scores are the softmax over all outputs, the choice is by score +
// correction within the `keep` best of `groups` equal groups (a group's score:
// its largest choice), weights are the scores. Else by logit, weights are the
// softmax over the chosen logits.
struct Routing {
  const float* correction;  // null: none
  int E;         // outputs that can be chosen
  int real;      // experts with weights; those behind are identities
  int shared;    // slots of shared experts, behind the chosen ones
  int top, groups, keep;
  bool over_all;
  // router row E: gate of the shared experts
  __host__ __device__ int rows() const { return E + (shared > 0 ? 1 : 0); }
  __host__ __device__ int slots() const { return top + shared; }
  __host__ __device__ int plan() const { return real + shared; }
};

// One token's logits z [E] -> scores s = softmax, choices (in z's place), by
// one wave. gmax: a float per group.
__device__ __forceinline__ void choice_scores(float* z, float* s, float* gmax,
                                              const Routing& how, int EP) {
  const int lane = threadIdx.x & 63, E = how.E;
  float mx = -INFINITY;
  for (int e = lane; e < E; e += 64) mx = fmaxf(mx, z[e]);
  mx = wave_reduce_max(mx);
  float sum = 0.f;
  for (int e = lane; e < E; e += 64) {
    s[e] = expf(z[e] - mx);
    sum += s[e];
  }
  sum = wave_reduce_sum(sum);
  for (int e = lane; e < E; e += 64) {
    s[e] /= sum;
    z[e] = s[e] + (how.correction ? how.correction[e] : 0.f);
  }
  wave_lds_fence();
  if (how.keep >= how.groups) return;
  const int size = E / how.groups;
  for (int q = lane; q < how.groups; q += 64) {
    float m = -INFINITY;
    for (int e = q * size; e < (q + 1) * size; ++e) m = fmaxf(m, z[e]);
    gmax[q] = m;
  }
  wave_lds_fence();
  for (int e = lane; e < E; e += 64) {
    const int q = e / size;
    const float mine = gmax[q];
    int place = 0;
    for (int j = 0; j < how.groups; ++j)
      place += gmax[j] > mine || (gmax[j] == mine && j < q);
    if (place >= how.keep) z[e] = -INFINITY;
  }
  wave_lds_fence();
}

// Logits in float, the `top` best (ties: the lower expert), their weights.
// Counts per expert and each slot's rank in it for the grouping; a single
// workgroup groups right away. KW: waves, which split the inner dimension.
template <typename T, int KW>
__global__ __launch_bounds__(KW * 64) void moe_route_kernel(
    const T* __restrict__ h, const T* __restrict__ router, int n_tok, int K,
    Routing how, float* __restrict__ share, int* __restrict__ ids,
    int* __restrict__ rank, int* __restrict__ counts, int* __restrict__ pos,
    int* __restrict__ tok, int rows, int* __restrict__ tiles,
    int* __restrict__ n_tiles) {
  constexpr int NTH = KW * 64;
  constexpr int PER = RT * MAX_TOP / NTH;  // most slots of a thread
  __shared__ __align__(16) float part[KW][RT][64 + 4];
  __shared__ float gate[RT];
  extern __shared__ __align__(16) char smem[];
  const int E = how.E, top = how.top, NR = how.rows(), PE = how.plan();
  const int TS = how.slots();
  const int EP = (E + 3) & ~3;
  float* logits = (float*)smem;            // [RT][EP]
  float* best = logits + RT * EP;          // [RT][top]
  int* chosen = (int*)(best + RT * top);   // [RT][top]
  int* cnt = chosen + RT * top;            // [PE]
  int* off = cnt + PE;                     // [PE]
  float* score = (float*)(off + PE);       // [RT][EP] if over_all
  float* group = score + RT * EP;          // [KW][groups] if over_all
  const int tid = threadIdx.x, lane = tid & 63, wave = uniform_wave();
  const int r16 = lane & 15, ko = (lane >> 4) * 8;
  const int t0 = blockIdx.x * RT;
  const int nt = min(RT, n_tok - t0);
  for (int e = tid; e < PE; e += NTH) cnt[e] = 0;
  // whatever the logits are (nan), every slot has an expert
  for (int i = tid; i < RT * top; i += NTH) {
    chosen[i] = i % top;
    best[i] = 0.f;
  }

  const T* hr = h + (long)min(t0 + r16, n_tok - 1) * K + ko;
  const int steps = K / 32, per = (steps + KW - 1) / KW;
  const int k_lo = wave * per * 32, k_hi = min(K, k_lo + per * 32);
  for (int e0 = 0; e0 < NR; e0 += 64) {
    const T* wr = router + ko;
    if (NR - e0 <= 16)
      router_tiles<T, 1>(hr, wr, e0, NR, K, k_lo, k_hi, &part[wave][r16][0]);
    else if (NR - e0 <= 32)
      router_tiles<T, 2>(hr, wr, e0, NR, K, k_lo, k_hi, &part[wave][r16][0]);
    else
      router_tiles<T, 4>(hr, wr, e0, NR, K, k_lo, k_hi, &part[wave][r16][0]);
    __syncthreads();
    for (int i = tid; i < RT * 64; i += NTH) {
      const int t = i >> 6, e = e0 + (i & 63);
      float s = 0.f;
#pragma unroll
      for (int w = 0; w < KW; ++w) s += part[w][t][i & 63];
      if (e < EP) logits[t * EP + e] = e < E ? s : -INFINITY;
      if (e == E && NR > E) gate[t] = 1.f / (1.f + expf(-s));
    }
    __syncthreads();
  }

  // an expert's place is the number of experts in front of it
  for (int t = wave; t < nt; t += KW) {
    float* z = logits + t * EP;
    if (how.over_all)
      choice_scores(z, score + t * EP, group + wave * how.groups, how, EP);
    for (int e = lane; e < E; e += 64) {
      const float mine = z[e];
      int place = 0;
#pragma unroll 4
      for (int j = 0; j < EP; j += 4) {
        const lm_f32x4 o = *reinterpret_cast<const lm_f32x4*>(z + j);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          place += o[r] > mine || (o[r] == mine && j + r < e);
      }
      if (place < top) {
        chosen[t * top + place] = e;
        best[t * top + place] = how.over_all ? score[t * EP + e] : mine;
      }
    }
    wave_lds_fence();
    float v = lane < top ? best[t * top + lane] : 0.f;
    if (!how.over_all) {
      v = lane < top ? expf(v - best[t * top]) : 0.f;
      v /= wave_reduce_sum(v);
    }
    if (lane >= top) v = gate[t];
    if (lane < TS) share[(long)(t0 + t) * TS + lane] = v;
  }
  __syncthreads();
  const bool alone = gridDim.x == 1;
  // a slot's expert in the plan, -1: an identity
  auto plan_expert = [&](int s) {
    const int k = s % TS;
    if (k >= top) return how.real + k - top;
    const int e = chosen[s / TS * top + k];
    return e < how.real ? e : -1;
  };
  int rk[PER];
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int s = tid + j * NTH;
    rk[j] = 0;
    if (s < nt * TS) {
      const int e = plan_expert(s);
      if (e >= 0) rk[j] = atomicAdd(&cnt[e], 1);
      if (!alone) {
        ids[(long)t0 * TS + s] = e;
        rank[(long)t0 * TS + s] = rk[j];
      }
    }
  }
  __syncthreads();
  if (!alone) {
    for (int e = tid; e < PE; e += NTH)
      counts[(long)blockIdx.x * PE + e] = cnt[e];
    return;
  }
  scan_experts(cnt, off, PE, rows, tiles, n_tiles);
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int s = tid + j * NTH;
    if (s < nt * TS) {
      const int e = plan_expert(s);
      const int p = e < 0 ? -1 : off[e] + rk[j];
      pos[s] = p;
      if (p >= 0) tok[p] = s / TS;
    }
  }
}

// workgroup b puts the slots of routing workgroup b into their rows
__global__ __launch_bounds__(256) void moe_place_kernel(
    const int* __restrict__ ids, const int* __restrict__ rank,
    const int* __restrict__ counts, int n_wg, int n_tok, int E, int top,
    int* __restrict__ pos, int* __restrict__ tok, int rows,
    int* __restrict__ tiles, int* __restrict__ n_tiles) {
  extern __shared__ __align__(16) char smem[];
  int* tot = (int*)smem;   // [E] all workgroups
  int* bef = tot + E;      // [E] those in front of this one
  int* off = bef + E;      // [E]
  const int tid = threadIdx.x, b = blockIdx.x;
  for (int e = tid; e < E; e += 256) tot[e] = bef[e] = 0;
  __syncthreads();
  const int groups = max(1, 256 / E);
  for (int i = tid; i < groups * E; i += 256) {
    const int e = i % E, g = i / E;
    int all = 0, front = 0;
#pragma unroll 8
    for (int w = g; w < n_wg; w += groups) {
      const int c = counts[(long)w * E + e];
      all += c;
      front += w < b ? c : 0;
    }
    atomicAdd(&tot[e], all);
    atomicAdd(&bef[e], front);
  }
  __syncthreads();
  scan_experts(tot, off, E, rows, b == 0 ? tiles : nullptr, n_tiles);
  const int n = min(RT, n_tok - b * RT) * top;
  for (int i = tid; i < n; i += 256) {
    const long s = (long)b * RT * top + i;
    const int e = ids[s];
    const int p = e < 0 ? -1 : off[e] + bef[e] + rank[s];
    pos[s] = p;
    if (p >= 0) tok[p] = (int)(s / top);
  }
}

// Four neighbouring columns of a product, behind their activation. A gated one
// (LM_SWIGLU) takes columns in pairs (gate, up) and makes one of each.
template <int ACT> __host__ __device__ constexpr long out_cols(long n) {
  return ACT == LM_SWIGLU ? n / 2 : n;
}
__device__ __forceinline__ void store2(bf16* p, float a, float b) {
  union { unsigned u; bf16 h[2]; } o;
  o.h[0] = __float2bfloat16(a);
  o.h[1] = __float2bfloat16(b);
  *reinterpret_cast<unsigned*>(p) = o.u;
}
__device__ __forceinline__ void store2(float* p, float a, float b) {
  *reinterpret_cast<float2*>(p) = float2{a, b};
}
template <typename T, int ACT>
__device__ __forceinline__ void store_act(T* p, const lm_f32x4& s) {
  if (ACT == LM_SWIGLU) {
    store2(p, act_f<LM_SILU>(s[0]) * s[1], act_f<LM_SILU>(s[2]) * s[3]);
  } else {
    const float f[4] = {act_f<ACT>(s[0]), act_f<ACT>(s[1]), act_f<ACT>(s[2]),
                        act_f<ACT>(s[3])};
    store4(p, f);
  }
}

// ------------------------------------------------------------------- //
// grouped product, few rows per expert: 16 * NT columns and up to 16 * MT rows
// per workgroup, operands straight from memory, waves split the inner
// dimension
// ------------------------------------------------------------------- //
constexpr int GW = 8;

template <typename T, int MT, int NT, int ACT>
__global__ __launch_bounds__(GW * 64) void moe_rows_kernel(
    const T* __restrict__ a, const int* __restrict__ tok,  // null: row = row
    const T* __restrict__ w, T* __restrict__ out,
    const int* __restrict__ tiles, const int* __restrict__ n_tiles, int N,
    int K, int n_rows, int n_a) {
  __shared__ __align__(16) float part[GW][MT * 16][NT * 16 + 4];
  if ((int)blockIdx.y >= n_tiles[0]) return;
  const int* td = tiles + (long)blockIdx.y * 3;
  const int e = td[0], r0 = td[1], cnt = td[2];
  const int n0 = blockIdx.x * (NT * 16);
  const int tid = threadIdx.x, lane = tid & 63, wave = uniform_wave();
  const int r16 = lane & 15, g = lane >> 4, ko = g * 8;
  const T* wr[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i)
    wr[i] = w + ((long)e * N + n0 + i * 16 + r16) * K + ko;
  const T* ar[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const int p = min(r0 + min(i * 16 + r16, cnt - 1), n_rows - 1);
    const int row = tok ? tok[p] : p;
    ar[i] = a + (long)min(row, n_a - 1) * K + ko;
  }
  lm_f32x4 acc[MT][NT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[i][j] = lm_f32x4{0.f, 0.f, 0.f, 0.f};
  const int per = (K / 32 + GW - 1) / GW;
  const int k_lo = wave * per * 32, k_hi = min(K, k_lo + per * 32);
  // U steps of operands in registers, the next U on their way
  constexpr int U = 4;
  Frag<T> wf[2][U][NT], af[2][U][MT];
  auto load = [&](int b, int k0) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + u * 32;
      if (k < k_hi) {
#pragma unroll
        for (int j = 0; j < NT; ++j) wf[b][u][j] = load_frag(wr[j] + k);
#pragma unroll
        for (int i = 0; i < MT; ++i) af[b][u][i] = load_frag(ar[i] + k);
      }
    }
  };
  auto multiply = [&](int b, int k0) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (k0 + u * 32 < k_hi) {
#pragma unroll
        for (int i = 0; i < MT; ++i)
#pragma unroll
          for (int j = 0; j < NT; ++j)
            acc[i][j] = mma32(wf[b][u][j], af[b][u][i], acc[i][j]);
      }
    }
  };
  load(0, k_lo);
  for (int k = k_lo; k < k_hi; k += 2 * U * 32) {
    load(1, k + U * 32);
    multiply(0, k);
    load(0, k + 2 * U * 32);
    multiply(1, k + U * 32);
  }
#pragma unroll
  for (int i = 0; i < MT; ++i) {
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      const float f[4] = {acc[i][j][0], acc[i][j][1], acc[i][j][2],
                          acc[i][j][3]};
      store4(&part[wave][i * 16 + r16][j * 16 + 4 * g], f);
    }
  }
  __syncthreads();
  for (int i = tid; i < MT * NT * 64; i += GW * 64) {
    const int m = i / (NT * 4), c = (i % (NT * 4)) * 4;
    if (m >= cnt) break;
    lm_f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int v = 0; v < GW; ++v)
      s += *reinterpret_cast<const lm_f32x4*>(&part[v][m][c]);
    store_act<T, ACT>(out + (long)(r0 + m) * out_cols<ACT>(N) +
                          out_cols<ACT>(n0 + c), s);
  }
}

// ------------------------------------------------------------------- //
// grouped product on BM x BN tiles (bf16): inner steps of 64 through NS LDS
// buffers filled by direct-to-LDS loads
// ------------------------------------------------------------------- //
// The loads write LDS in lane order, so the 16-byte pieces of a row are
// permuted by (row & 7) at the source and again at the read: fragment reads
// touch all banks. The weights are the first MFMA operand: a lane then holds
// four neighbouring columns of one row of the result. One barrier per step:
// it says that step i's buffer is full and that everyone is done with step
// i - 1's, which is filled next.
constexpr int BK = 64;

// Direct-to-LDS load of 16 bytes per lane, lane l to lds + 16 l. As assembly:
// the compiler would wait for all of them in front of every LDS read, since it
// cannot tell the buffers apart. wait_loads says when a step has landed.
__device__ __forceinline__ void load_to_lds(const bf16* src, unsigned lds) {
  asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\t"
               "global_load_lds_dwordx4 %1, off"
               ::"s"(lds), "v"(src)
               : "m0", "memory");
}
// until at most N of the wave's loads are in flight
template <int N> __device__ __forceinline__ void wait_loads() {
  static_assert(N < 64, "six bits");
  asm volatile("s_waitcnt vmcnt(%0)" ::"n"(N) : "memory");
}
__device__ __forceinline__ unsigned lds_address(const void* p) {
  return (unsigned)(size_t)(__attribute__((address_space(3))) const char*)p;
}

template <int BM, int BN, int WM, int WN, int NS, int ACT>
__global__ __launch_bounds__(WM * WN * 64,
                             NS * BK * (BM + BN) * 2 > 80 * 1024
                                 ? WM * WN / 4 : WM * WN / 2)
void moe_tile_kernel(
    const bf16* __restrict__ a, const int* __restrict__ tok,
    const bf16* __restrict__ w, bf16* __restrict__ out,
    const int* __restrict__ tiles, const int* __restrict__ n_tiles, int N,
    int K, int n_rows, int n_a) {
  constexpr int NTH = WM * WN * 64;
  constexpr int FM = BM / WM / 16, FN = BN / WN / 16;
  constexpr int IA = BM * 8 / NTH, IB = BN * 8 / NTH;
  static_assert(IA * NTH == BM * 8 && IB * NTH == BN * 8, "whole pieces");
  __shared__ __align__(16) short la[NS][BM * BK];
  __shared__ __align__(16) short lb[NS][BN * BK];
  const int nb = (N + BN - 1) / BN;
  const int nwg = n_tiles[0] * nb;
  if ((int)blockIdx.x >= nwg) return;
  // workgroup b runs on XCD b % 8: give each XCD neighbouring tiles, which
  // share rows (same tile) and weights (same expert) in its L2
  const int xcd = blockIdx.x % 8, idx = blockIdx.x / 8;
  const int q8 = nwg / 8, r8 = nwg % 8;
  const int bid = xcd * q8 + min(xcd, r8) + idx;
  const int* td = tiles + (long)(bid / nb) * 3;
  const int e = td[0], r0 = td[1], cnt = td[2];
  const int n0 = (bid % nb) * BN;
  const int tid = threadIdx.x, lane = tid & 63, wave = uniform_wave();
  const int r16 = lane & 15, g = lane >> 4;
  const int wm = (wave / WN) * (BM / WM), wn = (wave % WN) * (BN / WN);

  // a thread's pieces: row (i * NTH + tid) / 8, LDS piece tid % 8
  const int piece = ((tid & 7) ^ ((tid >> 3) & 7)) * 8;
  const bf16* pa[IA];
  const bf16* pb[IB];
#pragma unroll
  for (int i = 0; i < IA; ++i) {
    const int r = min((i * NTH + tid) >> 3, cnt - 1);
    const int p = min(r0 + r, n_rows - 1);
    const int row = tok ? tok[p] : p;
    pa[i] = a + (long)min(row, n_a - 1) * K + piece;
  }
#pragma unroll
  for (int i = 0; i < IB; ++i) {
    const int n = min(n0 + ((i * NTH + tid) >> 3), N - 1);
    pb[i] = w + ((long)e * N + n) * K + piece;
  }
  const unsigned a_lds = lds_address(la) + wave * 1024;
  const unsigned b_lds = lds_address(lb) + wave * 1024;
  auto stage = [&](int buf, int k) {
#pragma unroll
    for (int i = 0; i < IB; ++i)
      load_to_lds(pb[i] + k, b_lds + (buf * BN * 8 + i * NTH) * 16);
#pragma unroll
    for (int i = 0; i < IA; ++i)
      load_to_lds(pa[i] + k, a_lds + (buf * BM * 8 + i * NTH) * 16);
  };

  lm_f32x4 acc[FN][FM];
#pragma unroll
  for (int i = 0; i < FN; ++i)
#pragma unroll
    for (int j = 0; j < FM; ++j) acc[i][j] = lm_f32x4{0.f, 0.f, 0.f, 0.f};

  // Steps behind the last one load the last step's pieces again, into a
  // buffer that nobody reads any more: the count of loads in flight stays
  // the same for every step. All have landed before the workgroup ends.
  const int last = K - BK;
#pragma unroll
  for (int i = 0; i < NS - 1; ++i) stage(i, min(i * BK, last));
  int cur = 0;
  for (int k = 0; k < K; k += BK) {
    wait_loads<(NS - 2) * (IA + IB)>();
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    if (NS > 2 || k + BK < K)
      stage(cur == 0 ? NS - 1 : cur - 1, min(k + (NS - 1) * BK, last));
#pragma unroll
    for (int kc = 0; kc < 2; ++kc) {
      const int s = ((kc * 4 + g) ^ (r16 & 7)) * 8;
      lm_s16x8 fa[FM], fb[FN];
#pragma unroll
      for (int j = 0; j < FM; ++j)
        fa[j] = *reinterpret_cast<const lm_s16x8*>(
            &la[cur][(wm + j * 16 + r16) * BK + s]);
#pragma unroll
      for (int i = 0; i < FN; ++i)
        fb[i] = *reinterpret_cast<const lm_s16x8*>(
            &lb[cur][(wn + i * 16 + r16) * BK + s]);
      __builtin_amdgcn_s_setprio(1);
#pragma unroll
      for (int i = 0; i < FN; ++i)
#pragma unroll
        for (int j = 0; j < FM; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              fb[i], fa[j], acc[i][j], 0, 0, 0);
      __builtin_amdgcn_s_setprio(0);
    }
    cur = cur == NS - 1 ? 0 : cur + 1;
  }
  wait_loads<0>();

#pragma unroll
  for (int j = 0; j < FM; ++j) {
    const int m = wm + j * 16 + r16;
    if (m < cnt) {
      bf16* dst = out + (long)(r0 + m) * out_cols<ACT>(N) +
                  out_cols<ACT>(n0 + wn + 4 * g);
#pragma unroll
      for (int i = 0; i < FN; ++i) {
        if (n0 + wn + i * 16 < N)
          store_act<bf16, ACT>(dst + out_cols<ACT>(i * 16), acc[i][j]);
      }
    }
  }
}

// most tiles that S slots over E experts can make
long max_tiles(long S, long E, long rows) {
  return std::min(S, S / rows + std::min(E, S));
}

}  // namespace

// Without `correction` and groups (0): the `top` largest logits, weighed by the
// softmax over them. router [choices (+ 1 gate row with shared slots), K].
// -> {share float [T, slots], pos int [T, slots], tok int [T * slots],
//     plan int [1 + 3 * tiles]: the number of tiles, then (expert, first row,
//     rows) each}; slots = top + shared
std::vector<torch::Tensor> lm_moe_route(torch::Tensor h, torch::Tensor router,
                                        long top, long rows, bool over_all,
                                        c10::optional<torch::Tensor> correction,
                                        long groups, long keep, long identity,
                                        long shared) {
  LM_CHECK_CONTIG(h);
  LM_CHECK_CONTIG(router);
  TORCH_CHECK(h.dim() == 2 && router.dim() == 2 &&
              h.size(1) == router.size(1) &&
              h.scalar_type() == router.scalar_type());
  Routing how{};
  how.E = (int)router.size(0) - (shared > 0 ? 1 : 0);
  how.real = how.E - (int)identity;
  how.shared = (int)shared;
  how.top = (int)top;
  how.groups = (int)groups;
  how.keep = (int)keep;
  how.over_all = over_all;
  const int T = h.size(0), K = h.size(1), E = how.E, PE = how.plan();
  const int slots = how.slots();
  TORCH_CHECK(K % 32 == 0 && E >= 1 && E <= 1024 && PE <= 1024,
              "lm_moe_route: sizes");
  TORCH_CHECK(top >= 1 && slots <= MAX_TOP && top <= E && rows >= 1);
  TORCH_CHECK(identity >= 0 && shared >= 0 && PE >= 1 && how.real >= 0);
  TORCH_CHECK(groups >= 1 && keep >= 1 && keep <= groups && E % groups == 0,
              "lm_moe_route: groups");
  TORCH_CHECK(over_all || (groups == 1 && !correction));
  if (correction) {
    TORCH_CHECK(correction->is_cuda() && correction->is_contiguous() &&
                correction->numel() == E &&
                correction->scalar_type() == at::kFloat);
    how.correction = correction->data_ptr<float>();
  }
  TORCH_CHECK((long)T * slots < (1L << 30));
  auto i32 = h.options().dtype(at::kInt);
  const long S = (long)T * slots;
  auto share = torch::empty({T, slots}, h.options().dtype(at::kFloat));
  auto pos = torch::empty({T, slots}, i32);
  auto tok = torch::empty({S}, i32);
  auto plan = torch::empty({1 + 3 * max_tiles(S, PE, rows)}, i32);
  if (T == 0) return {share, pos, tok, plan};
  const int n_wg = (T + RT - 1) / RT;
  torch::Tensor ids, rank, counts;
  if (n_wg > 1) {
    ids = torch::empty({S}, i32);
    rank = torch::empty({S}, i32);
    counts = torch::empty({n_wg, PE}, i32);
  }
  int* pp = plan.data_ptr<int>();
  hipStream_t st = cmls::current_stream();
#define LM_MRT(KW)                                                           \
  do {                                                                       \
    const int ep = (E + 3) & ~3;                                             \
    const int bytes =                                                        \
        (RT * (ep + 2 * (int)top) + 2 * PE +                                 \
         (over_all ? RT * ep + KW * (int)groups : 0)) * 4;                   \
    TORCH_CHECK(bytes + KW * RT * 68 * 4 + 8192 <= 160 * 1024,               \
                "lm_moe_route: ", E, " outputs do not fit LDS");             \
    auto* fn = &moe_route_kernel<scalar_t, KW>;                              \
    HIP_CHECK(hipFuncSetAttribute(                                           \
        reinterpret_cast<const void*>(fn),                                   \
        hipFuncAttributeMaxDynamicSharedMemorySize, bytes));                 \
    hipLaunchKernelGGL(fn, dim3(n_wg), dim3(KW * 64), bytes, st,             \
                       (const scalar_t*)h.data_ptr(),                        \
                       (const scalar_t*)router.data_ptr(), T, K, how,        \
                       share.data_ptr<float>(),                              \
                       n_wg > 1 ? ids.data_ptr<int>() : nullptr,             \
                       n_wg > 1 ? rank.data_ptr<int>() : nullptr,            \
                       n_wg > 1 ? counts.data_ptr<int>() : nullptr,          \
                       pos.data_ptr<int>(), tok.data_ptr<int>(), (int)rows,  \
                       pp + 1, pp);                                          \
  } while (0)
  LM_DISPATCH(h, "lm_moe_route", [&] {
    if (n_wg <= 256) LM_MRT(16);  // few workgroups: short chains of loads
    else LM_MRT(8);
  });
#undef LM_MRT
  LM_LAUNCHED();
  if (n_wg > 1) {
    hipLaunchKernelGGL(moe_place_kernel, dim3(n_wg), dim3(256),
                       3 * PE * 4, st, ids.data_ptr<int>(),
                       rank.data_ptr<int>(), counts.data_ptr<int>(), n_wg, T,
                       PE, slots, pos.data_ptr<int>(), tok.data_ptr<int>(),
                       (int)rows, pp + 1, pp);
    LM_LAUNCHED();
  }
  return {share, pos, tok, plan};
}

// out[r] = act(w[expert of r] @ a[tok[r]]); w [E, N, K]; tok absent: a[r].
// LM_SWIGLU: rows of w in pairs (gate, up), out has N / 2 columns.
// `rows`: rows per tile that the plan was made for
torch::Tensor lm_moe_gemm(torch::Tensor a, c10::optional<torch::Tensor> tok,
                          torch::Tensor w, torch::Tensor plan, long n_rows,
                          long rows, long act) {
  LM_CHECK_CONTIG(a);
  LM_CHECK_CONTIG(w);
  LM_CHECK_I32(plan);
  TORCH_CHECK(a.dim() == 2 && w.dim() == 3 && a.size(1) == w.size(2) &&
              a.scalar_type() == w.scalar_type());
  const int E = w.size(0), N = w.size(1), K = w.size(2);
  TORCH_CHECK(N % 32 == 0 && K % 32 == 0, "lm_moe_gemm: sizes");
  TORCH_CHECK(act == LM_RELU2 || act == LM_NO_ACT || act == LM_SWIGLU);
  if (tok) {
    LM_CHECK_I32(*tok);
    TORCH_CHECK(tok->numel() == n_rows);
  } else {
    TORCH_CHECK(a.size(0) == n_rows);
  }
  const long nt = max_tiles(n_rows, E, rows);
  TORCH_CHECK(plan.numel() == 1 + 3 * nt, "lm_moe_gemm: plan for other rows");
  auto out = torch::empty({n_rows, act == LM_SWIGLU ? N / 2 : N},
                          a.options());
  if (n_rows == 0) return out;
  TORCH_CHECK(a.size(0) > 0);
  hipStream_t st = cmls::current_stream();
  const int* pp = plan.data_ptr<int>();
  const int* tk = tok ? tok->data_ptr<int>() : nullptr;
#define LM_MG_ARGS(TY)                                                      \
  (const TY*)a.data_ptr(), tk, (const TY*)w.data_ptr(), (TY*)out.data_ptr(),\
      pp + 1, pp, N, K, (int)n_rows, (int)a.size(0)
  if (rows != 16 && a.scalar_type() == at::kBFloat16 && K % BK == 0) {
#define LM_MT(BM, BN, WM, WN, NS, ACT)                                      \
  do {                                                                      \
    const long wgs = nt * ((N + BN - 1) / BN);                              \
    TORCH_CHECK(wgs < (1L << 31));                                          \
    hipLaunchKernelGGL((moe_tile_kernel<BM, BN, WM, WN, NS, ACT>),          \
                       dim3(wgs), dim3(WM * WN * 64), 0, st,                \
                       LM_MG_ARGS(bf16));                                   \
  } while (0)
#define LM_MT_ACT(BM, BN, WM, WN, NS)                                       \
  do {                                                                      \
    if (act == LM_RELU2) LM_MT(BM, BN, WM, WN, NS, LM_RELU2);               \
    else if (act == LM_SWIGLU) LM_MT(BM, BN, WM, WN, NS, LM_SWIGLU);        \
    else LM_MT(BM, BN, WM, WN, NS, LM_NO_ACT);                              \
  } while (0)
    if (rows == 256) LM_MT_ACT(256, 256, 2, 4, 2);
    else if (rows == 128) LM_MT_ACT(128, 128, 2, 2, 2);
    else if (rows == 64) LM_MT_ACT(64, 64, 2, 2, 4);
    else if (rows == 32) LM_MT_ACT(32, 64, 1, 4, 4);
    else TORCH_CHECK(false, "lm_moe_gemm: rows per tile");
#undef LM_MT_ACT
#undef LM_MT
  } else {
    TORCH_CHECK(nt <= 65535);
#define LM_MR(MT, NT, ACT)                                                  \
  hipLaunchKernelGGL((moe_rows_kernel<scalar_t, MT, NT, ACT>),              \
                     dim3(N / (16 * NT), nt), dim3(GW * 64), 0, st,         \
                     LM_MG_ARGS(scalar_t))
#define LM_MR_ACT(MT, NT)                                                   \
  do {                                                                      \
    if (act == LM_RELU2) LM_MR(MT, NT, LM_RELU2);                           \
    else if (act == LM_SWIGLU) LM_MR(MT, NT, LM_SWIGLU);                    \
    else LM_MR(MT, NT, LM_NO_ACT);                                          \
  } while (0)
    LM_DISPATCH(a, "lm_moe_gemm", [&] {
      if (rows == 16) LM_MR_ACT(1, 1);
      else if (rows == 64) LM_MR_ACT(4, 2);
      else TORCH_CHECK(false, "lm_moe_gemm: rows per tile");
    });
#undef LM_MR_ACT
#undef LM_MR
  }
#undef LM_MG_ARGS
  LM_LAUNCHED();
  return out;
}
