// Mixture of experts on a flat token batch: routing, grouping by expert and
// the grouped products.
//
// Every token takes `top` experts. Its T * top slots are put in expert order
// (pos: slot -> row, tok: row -> token); a tile list cuts each expert's rows
// into pieces of at most `rows` rows. A grouped product runs one workgroup per
// (tile, column range) and takes its row count from the list, so nothing is
// read back to the host. The list's length lies in device memory: a launch
// covers the most tiles there can be and the surplus workgroups leave at once.
// A row's result does not depend on where its expert's rows end up.
#include "lm_common.h"

namespace {

constexpr int RT = 16;   // tokens per routing workgroup
constexpr int RW = 8;    // its waves; they split the inner dimension
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

// Logits in float, the `top` largest (ties: the lower expert), softmax over
// them. Counts per expert and each slot's rank in it for the grouping; a
// single workgroup groups right away.
template <typename T>
__global__ __launch_bounds__(RW * 64) void moe_route_kernel(
    const T* __restrict__ h, const T* __restrict__ router, int n_tok, int K,
    int E, int top, float* __restrict__ share, int* __restrict__ ids,
    int* __restrict__ rank, int* __restrict__ counts, int* __restrict__ pos,
    int* __restrict__ tok, int rows, int* __restrict__ tiles,
    int* __restrict__ n_tiles) {
  __shared__ __align__(16) float part[RW][RT][64 + 4];
  __shared__ int chosen[RT][MAX_TOP];
  extern __shared__ __align__(16) char smem[];
  float* logits = (float*)smem;         // [RT][E]
  int* cnt = (int*)(logits + RT * E);   // [E]
  int* off = cnt + E;                   // [E]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int r16 = lane & 15, g = lane >> 4, ko = g * 8;
  const int t0 = blockIdx.x * RT;
  const int nt = min(RT, n_tok - t0);
  for (int e = tid; e < E; e += RW * 64) cnt[e] = 0;

  const T* hr = h + (long)min(t0 + r16, n_tok - 1) * K + ko;
  const int steps = K / 32, per = (steps + RW - 1) / RW;
  const int k_lo = wave * per * 32, k_hi = min(K, k_lo + per * 32);
  for (int e0 = 0; e0 < E; e0 += 64) {
    lm_f32x4 acc[4];
    const T* wr[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      acc[i] = lm_f32x4{0.f, 0.f, 0.f, 0.f};
      wr[i] = router + (long)min(e0 + i * 16 + r16, E - 1) * K + ko;
    }
#pragma unroll 4
    for (int k = k_lo; k < k_hi; k += 32) {
      const Frag<T> hf = load_frag(hr + k);
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (e0 + i * 16 < E) acc[i] = mma32(load_frag(wr[i] + k), hf, acc[i]);
    }
    // result rows are experts 4g..4g+3 of a tile, columns tokens
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float f[4] = {acc[i][0], acc[i][1], acc[i][2], acc[i][3]};
      store4(&part[wave][r16][i * 16 + 4 * g], f);
    }
    __syncthreads();
    for (int i = tid; i < RT * 64; i += RW * 64) {
      const int t = i >> 6, e = i & 63;
      float s = 0.f;
#pragma unroll
      for (int w = 0; w < RW; ++w) s += part[w][t][e];
      if (e0 + e < E) logits[t * E + e0 + e] = s;
    }
    __syncthreads();
  }

  for (int t = wave; t < nt; t += RW) {
    float* z = logits + t * E;
    float mine = 0.f, first = 0.f;
    int my_id = 0;
    for (int k = 0; k < top; ++k) {
      float best = -INFINITY;
      int at = E - 1;
      for (int e = lane; e < E; e += 64)
        if (z[e] > best) { best = z[e]; at = e; }
#pragma unroll
      for (int d = 32; d > 0; d >>= 1) {
        const float b = __shfl_xor(best, d, 64);
        const int i = __shfl_xor(at, d, 64);
        if (b > best || (b == best && i < at)) { best = b; at = i; }
      }
      if (k == 0) first = best;
      if (lane == k) { mine = best; my_id = at; }
      if (lane == 0) z[at] = -INFINITY;
      wave_lds_fence();
    }
    const float e = lane < top ? expf(mine - first) : 0.f;
    const float sum = wave_reduce_sum(e);
    if (lane < top) {
      share[(long)(t0 + t) * top + lane] = e / sum;
      chosen[t][lane] = my_id;
    }
  }
  __syncthreads();
  const bool alone = gridDim.x == 1;
  int rk[RT * MAX_TOP / (RW * 64)];
#pragma unroll
  for (int j = 0; j < RT * MAX_TOP / (RW * 64); ++j) {
    const int s = tid + j * RW * 64;
    rk[j] = 0;
    if (s < nt * top) {
      const int e = chosen[s / top][s % top];
      rk[j] = atomicAdd(&cnt[e], 1);
      if (!alone) {
        ids[(long)t0 * top + s] = e;
        rank[(long)t0 * top + s] = rk[j];
      }
    }
  }
  __syncthreads();
  if (!alone) {
    for (int e = tid; e < E; e += RW * 64)
      counts[(long)blockIdx.x * E + e] = cnt[e];
    return;
  }
  scan_experts(cnt, off, E, rows, tiles, n_tiles);
#pragma unroll
  for (int j = 0; j < RT * MAX_TOP / (RW * 64); ++j) {
    const int s = tid + j * RW * 64;
    if (s < nt * top) {
      const int p = off[chosen[s / top][s % top]] + rk[j];
      pos[s] = p;
      tok[p] = s / top;
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
    const int p = off[e] + bef[e] + rank[s];
    pos[s] = p;
    tok[p] = (int)(s / top);
  }
}

// ------------------------------------------------------------------- //
// grouped product, few rows per expert: 16 columns and up to 16 * MT rows per
// workgroup, operands straight from memory, waves split the inner dimension
// ------------------------------------------------------------------- //
constexpr int GW = 8;

template <typename T, int MT, int ACT>
__global__ __launch_bounds__(GW * 64) void moe_rows_kernel(
    const T* __restrict__ a, const int* __restrict__ tok,  // null: row = row
    const T* __restrict__ w, T* __restrict__ out,
    const int* __restrict__ tiles, const int* __restrict__ n_tiles, int N,
    int K, int n_rows, int n_a) {
  __shared__ __align__(16) float part[GW][MT][16][16 + 4];
  if ((int)blockIdx.y >= n_tiles[0]) return;
  const int* td = tiles + (long)blockIdx.y * 3;
  const int e = td[0], r0 = td[1], cnt = td[2];
  const int n0 = blockIdx.x * 16;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int r16 = lane & 15, g = lane >> 4, ko = g * 8;
  const T* wr = w + ((long)e * N + n0 + r16) * K + ko;
  const T* ar[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const int p = min(r0 + min(i * 16 + r16, cnt - 1), n_rows - 1);
    const int row = tok ? tok[p] : p;
    ar[i] = a + (long)min(row, n_a - 1) * K + ko;
  }
  lm_f32x4 acc[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i) acc[i] = lm_f32x4{0.f, 0.f, 0.f, 0.f};
  const int per = (K / 32 + GW - 1) / GW;
  const int k_lo = wave * per * 32, k_hi = min(K, k_lo + per * 32);
#pragma unroll 4
  for (int k = k_lo; k < k_hi; k += 32) {
    const Frag<T> wf = load_frag(wr + k);
#pragma unroll
    for (int i = 0; i < MT; ++i)
      acc[i] = mma32(wf, load_frag(ar[i] + k), acc[i]);
  }
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const float f[4] = {acc[i][0], acc[i][1], acc[i][2], acc[i][3]};
    store4(&part[wave][i][r16][4 * g], f);
  }
  __syncthreads();
  for (int i = tid; i < MT * 64; i += GW * 64) {
    const int m = i >> 2, c = (i & 3) * 4;
    if (m >= cnt) break;
    lm_f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int v = 0; v < GW; ++v)
      s += *reinterpret_cast<const lm_f32x4*>(&part[v][m >> 4][m & 15][c]);
    const float f[4] = {act_f<ACT>(s[0]), act_f<ACT>(s[1]), act_f<ACT>(s[2]),
                        act_f<ACT>(s[3])};
    store4(out + (long)(r0 + m) * N + n0 + c, f);
  }
}

// ------------------------------------------------------------------- //
// grouped product, many rows per expert (bf16): BM x BN tiles, inner steps of
// 64 through two LDS buffers filled by direct-to-LDS loads
// ------------------------------------------------------------------- //
// The loads write LDS in lane order, so the 16-byte pieces of a row are
// permuted by (row & 7) at the source and again at the read: fragment reads
// touch all banks. The weights are the first MFMA operand: a lane then holds
// four neighbouring columns of one row of the result.
constexpr int BK = 64;

template <int BM, int BN, int WM, int WN, int ACT>
__global__ __launch_bounds__(WM * WN * 64,
                             2 * BK * (BM + BN) * 2 > 80 * 1024
                                 ? WM * WN / 4 : WM * WN / 2)
void moe_tile_kernel(
    const bf16* __restrict__ a, const int* __restrict__ tok,
    const bf16* __restrict__ w, bf16* __restrict__ out,
    const int* __restrict__ tiles, const int* __restrict__ n_tiles, int N,
    int K, int n_rows, int n_a) {
  constexpr int NTH = WM * WN * 64;
  constexpr int FM = BM / WM / 16, FN = BN / WN / 16;
  constexpr int IA = BM * 8 / NTH, IB = BN * 8 / NTH;
  __shared__ __align__(16) short la[2][BM * BK];
  __shared__ __align__(16) short lb[2][BN * BK];
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
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
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
  auto stage = [&](int buf, int k) {
#pragma unroll
    for (int i = 0; i < IA; ++i)
      __builtin_amdgcn_global_load_lds(
          reinterpret_cast<const unsigned int*>(pa[i] + k),
          reinterpret_cast<unsigned int*>(&la[buf][(i * NTH + tid) * 8]), 16,
          0, 0);
#pragma unroll
    for (int i = 0; i < IB; ++i)
      __builtin_amdgcn_global_load_lds(
          reinterpret_cast<const unsigned int*>(pb[i] + k),
          reinterpret_cast<unsigned int*>(&lb[buf][(i * NTH + tid) * 8]), 16,
          0, 0);
  };

  lm_f32x4 acc[FN][FM];
#pragma unroll
  for (int i = 0; i < FN; ++i)
#pragma unroll
    for (int j = 0; j < FM; ++j) acc[i][j] = lm_f32x4{0.f, 0.f, 0.f, 0.f};

  stage(0, 0);
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  int cur = 0;
  for (int k = 0; k < K; k += BK) {
    if (k + BK < K) stage(cur ^ 1, k + BK);
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
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    cur ^= 1;
  }

#pragma unroll
  for (int j = 0; j < FM; ++j) {
    const int m = wm + j * 16 + r16;
    if (m < cnt) {
      bf16* dst = out + (long)(r0 + m) * N + n0 + wn + 4 * g;
#pragma unroll
      for (int i = 0; i < FN; ++i) {
        if (n0 + wn + i * 16 < N) {
          const float f[4] = {
              act_f<ACT>(acc[i][j][0]), act_f<ACT>(acc[i][j][1]),
              act_f<ACT>(acc[i][j][2]), act_f<ACT>(acc[i][j][3])};
          store4(dst + i * 16, f);
        }
      }
    }
  }
}

// most tiles that S slots over E experts can make
long max_tiles(long S, long E, long rows) {
  return std::min(S, S / rows + std::min(E, S));
}

}  // namespace

// -> {share float [T, top], pos int [T, top], tok int [T * top],
//     plan int [1 + 3 * tiles]: the number of tiles, then (expert, first row,
//     rows) each}
std::vector<torch::Tensor> lm_moe_route(torch::Tensor h, torch::Tensor router,
                                        long top, long rows) {
  LM_CHECK_CONTIG(h);
  LM_CHECK_CONTIG(router);
  TORCH_CHECK(h.dim() == 2 && router.dim() == 2 &&
              h.size(1) == router.size(1) &&
              h.scalar_type() == router.scalar_type());
  const int T = h.size(0), K = h.size(1), E = router.size(0);
  TORCH_CHECK(K % 32 == 0 && E >= 1 && E <= 1024, "lm_moe_route: sizes");
  TORCH_CHECK(top >= 1 && top <= MAX_TOP && top <= E && rows >= 1);
  TORCH_CHECK((long)T * top < (1L << 30));
  auto i32 = h.options().dtype(at::kInt);
  const long S = (long)T * top;
  auto share = torch::empty({T, top}, h.options().dtype(at::kFloat));
  auto pos = torch::empty({T, top}, i32);
  auto tok = torch::empty({S}, i32);
  auto plan = torch::empty({1 + 3 * max_tiles(S, E, rows)}, i32);
  if (T == 0) return {share, pos, tok, plan};
  const int n_wg = (T + RT - 1) / RT;
  torch::Tensor ids, rank, counts;
  if (n_wg > 1) {
    ids = torch::empty({S}, i32);
    rank = torch::empty({S}, i32);
    counts = torch::empty({n_wg, E}, i32);
  }
  int* pp = plan.data_ptr<int>();
  hipStream_t st = cmls::current_stream();
  LM_DISPATCH(h, "lm_moe_route", [&] {
    const int bytes = (RT * E + 2 * E) * 4;
    auto* fn = &moe_route_kernel<scalar_t>;
    HIP_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(fn),
                                  hipFuncAttributeMaxDynamicSharedMemorySize,
                                  bytes));
    hipLaunchKernelGGL(fn, dim3(n_wg), dim3(RW * 64), bytes, st,
                       (const scalar_t*)h.data_ptr(),
                       (const scalar_t*)router.data_ptr(), T, K, E, (int)top,
                       share.data_ptr<float>(),
                       n_wg > 1 ? ids.data_ptr<int>() : nullptr,
                       n_wg > 1 ? rank.data_ptr<int>() : nullptr,
                       n_wg > 1 ? counts.data_ptr<int>() : nullptr,
                       pos.data_ptr<int>(), tok.data_ptr<int>(), (int)rows,
                       pp + 1, pp);
  });
  LM_LAUNCHED();
  if (n_wg > 1) {
    hipLaunchKernelGGL(moe_place_kernel, dim3(n_wg), dim3(256), 3 * E * 4, st,
                       ids.data_ptr<int>(), rank.data_ptr<int>(),
                       counts.data_ptr<int>(), n_wg, T, E, (int)top,
                       pos.data_ptr<int>(), tok.data_ptr<int>(), (int)rows,
                       pp + 1, pp);
    LM_LAUNCHED();
  }
  return {share, pos, tok, plan};
}

// out[r] = act(w[expert of r] @ a[tok[r]]); w [E, N, K]; tok absent: a[r].
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
  TORCH_CHECK(act == LM_RELU2 || act == LM_NO_ACT);
  if (tok) {
    LM_CHECK_I32(*tok);
    TORCH_CHECK(tok->numel() == n_rows);
  } else {
    TORCH_CHECK(a.size(0) == n_rows);
  }
  const long nt = max_tiles(n_rows, E, rows);
  TORCH_CHECK(plan.numel() == 1 + 3 * nt, "lm_moe_gemm: plan for other rows");
  auto out = torch::empty({n_rows, N}, a.options());
  if (n_rows == 0) return out;
  TORCH_CHECK(a.size(0) > 0);
  hipStream_t st = cmls::current_stream();
  const int* pp = plan.data_ptr<int>();
  const int* tk = tok ? tok->data_ptr<int>() : nullptr;
#define LM_MG_ARGS(TY)                                                      \
  (const TY*)a.data_ptr(), tk, (const TY*)w.data_ptr(), (TY*)out.data_ptr(),\
      pp + 1, pp, N, K, (int)n_rows, (int)a.size(0)
  if (rows >= 128) {
    TORCH_CHECK(a.scalar_type() == at::kBFloat16 && K % BK == 0,
                "lm_moe_gemm: large tiles take bf16 and K % 64 == 0");
#define LM_MT(BM, BN, WM, WN, ACT)                                          \
  do {                                                                      \
    const long wgs = nt * ((N + BN - 1) / BN);                              \
    TORCH_CHECK(wgs < (1L << 31));                                          \
    hipLaunchKernelGGL((moe_tile_kernel<BM, BN, WM, WN, ACT>), dim3(wgs),   \
                       dim3(WM * WN * 64), 0, st, LM_MG_ARGS(bf16));        \
  } while (0)
#define LM_MT_ACT(BM, BN, WM, WN)                                           \
  do {                                                                      \
    if (act == LM_RELU2) LM_MT(BM, BN, WM, WN, LM_RELU2);                   \
    else LM_MT(BM, BN, WM, WN, LM_NO_ACT);                                  \
  } while (0)
    if (rows == 256) LM_MT_ACT(256, 256, 2, 4);
    else if (rows == 128) LM_MT_ACT(128, 128, 2, 2);
    else TORCH_CHECK(false, "lm_moe_gemm: 128 or 256 rows");
#undef LM_MT_ACT
#undef LM_MT
  } else {
    TORCH_CHECK(nt <= 65535);
#define LM_MR(MT, ACT)                                                      \
  hipLaunchKernelGGL((moe_rows_kernel<scalar_t, MT, ACT>), dim3(N / 16, nt),\
                     dim3(GW * 64), 0, st, LM_MG_ARGS(scalar_t))
#define LM_MR_ACT(MT)                                                       \
  do {                                                                      \
    if (act == LM_RELU2) LM_MR(MT, LM_RELU2);                               \
    else LM_MR(MT, LM_NO_ACT);                                              \
  } while (0)
    LM_DISPATCH(a, "lm_moe_gemm", [&] {
      if (rows == 16) LM_MR_ACT(1);
      else if (rows == 32) LM_MR_ACT(2);
      else if (rows == 64) LM_MR_ACT(4);
      else TORCH_CHECK(false, "lm_moe_gemm: 16, 32 or 64 rows");
    });
#undef LM_MR_ACT
#undef LM_MR
  }
#undef LM_MG_ARGS
  LM_LAUNCHED();
  return out;
}
