// Attention for prompt portions: flash attention on gathered rows, one per
// visible cached token of a sequence.
//
// - latent layers: keys and values were rebuilt per head from the cached
//   latents; per head a key is [nope part | rotated part], the rotated part is
//   shared by all heads and read from the gathered cache rows.
// - grouped layers: the gathered cache rows hold keys and values themselves, a
//   slice per key/value head.
//
// The workgroup takes 128 queries of one head (8 waves x 16) and walks the
// 64-key tiles that any of them can see. S^T = K Q^T leaves each lane with keys
// of ONE query, so max, sum and the running state are lane-local up to two
// shuffles; and because the k order of an MFMA is free, V is read (transposing
// LDS reads) in the key order that the S^T registers already have -- the
// weights go from registers straight into the second product.
#include "lm_attn.h"

namespace {

constexpr int BM = 128, BN = 64, NW = 8;

// Where a head's keys and values lie in the gathered rows. `per`: query heads
// per key/value head. A key is `kd` elements at k, the rest at rot. A layer
// whose values are its keys (SAME) has no v; its scores are multiplied by a
// float per row and key/value head.
struct PromptKeys {
  const bf16 *k, *rot, *v;
  const float* kscale;
  long k_row, rot_row, v_row, s_row;
  int k_head, v_head, kd, per;
};

struct PromptOut {
  const bf16* gate;  // [t, H*VP], null: none
  long ld_gate;
  bf16* out;
  long ld;           // out[t * ld + h * VP]
  float scale;
};

// qtiles: int32 [n, 6] = first token (flat), tokens, first position, first
// row in the gathered keys, what a row's number lacks to its position (rows
// behind the `keep` first ones), gathered rows. With `pool` [n, 7]: in the end
// the number of pooled rows, which stand first; row n is the mean of block n
// and is seen from position (n + 1) pool - 1 + window on.
// Two workgroups per CU (128 registers) where their LDS fits.
template <int QS, int VT, bool SAME>
__global__ __launch_bounds__(NW * 64, QS * 2 + VT <= 16 ? 4 : 2)
void prompt_attn_kernel(
    const bf16* __restrict__ q, long q_t,   // q[t * q_t + h * QD]
    PromptKeys src, const bf16* __restrict__ sink, PromptOut dst_,
    const int* __restrict__ qtiles, int H, int QD, int VP, int window,
    int keep, int pool, Score score) {
  constexpr int KP = QS * 32 + 8;   // LDS pitches
  constexpr int VPP = VT * 16 + 8;
  __shared__ __align__(16) short lk[2][BN * KP];
  __shared__ __align__(16) bf16 lv[2][SAME ? 8 : BN * VPP];
  __shared__ __align__(16) float ls[2][SAME ? BN : 4];
  // workgroup b runs on XCD b % 8: neighbouring heads, which share keys in
  // grouped layers, go to one XCD
  const int h = H % 8 ? blockIdx.x : blockIdx.x % 8 * (H / 8) + blockIdx.x / 8;
  const int hk = h / src.per;
  const int* td = qtiles + (long)blockIdx.y * (pool > 0 ? 7 : 6);
  const int t0 = td[0], len = td[1], p0 = td[2], kv0 = td[3], skip = td[4],
            nk = td[5];
  const int pooled = pool > 0 ? td[6] : 0;
  if (pool > 0) keep = pooled;
  auto place = [&](int n) {  // position that a row is seen from
    return n >= keep ? n + skip
                     : pool > 0 ? (n + 1) * pool - 1 + window : n;
  };
  const int tid = threadIdx.x, lane = tid & 63, wave = uniform_wave();
  const int r16 = lane & 15, g = lane >> 4, ko = g * 8;
  const int qrow = wave * 16 + r16;

  lm_s16x8 qf[QS];
#pragma unroll
  for (int kc = 0; kc < QS; ++kc) {
    qf[kc] = lm_s16x8{0, 0, 0, 0, 0, 0, 0, 0};
    if (qrow < len && kc * 32 < QD)
      qf[kc] = *reinterpret_cast<const lm_s16x8*>(
          q + (long)(t0 + qrow) * q_t + (long)h * QD + kc * 32 + ko);
  }
  float m_run = -INFINITY, l_run = 0.f;
  lm_f32x4 acc[VT];
#pragma unroll
  for (int i = 0; i < VT; ++i) acc[i] = lm_f32x4{0.f, 0.f, 0.f, 0.f};

  constexpr int KPC = (BN * QS * 4 + NW * 64 - 1) / (NW * 64);
  constexpr int VPC = (BN * VT * 2 + NW * 64 - 1) / (NW * 64);
  const int q8 = QD / 8, v8 = VP / 8;
  lm_s16x8 kreg[KPC], vreg[SAME ? 1 : VPC];
  float sreg = 0.f;
  auto stage_load = [&](int n0) {
#pragma unroll
    for (int i = 0; i < KPC; ++i) {
      const int p = tid + i * NW * 64;
      const int key = p / q8, d = (p % q8) * 8;
      kreg[i] = lm_s16x8{0, 0, 0, 0, 0, 0, 0, 0};
      if (key < BN && n0 + key < nk) {
        const long row = kv0 + n0 + key;
        kreg[i] = *reinterpret_cast<const lm_s16x8*>(
            d < src.kd ? src.k + row * src.k_row + hk * src.k_head + d
                       : src.rot + row * src.rot_row + (d - src.kd));
      }
    }
    if (SAME) {
      if (tid < BN)
        sreg = n0 + tid < nk ? src.kscale[(kv0 + n0 + tid) * src.s_row + hk]
                             : 0.f;
      return;
    }
#pragma unroll
    for (int i = 0; i < VPC; ++i) {
      const int p = tid + i * NW * 64;
      const int key = p / v8, d = (p % v8) * 8;
      vreg[SAME ? 0 : i] = lm_s16x8{0, 0, 0, 0, 0, 0, 0, 0};
      if (key < BN && n0 + key < nk)
        vreg[SAME ? 0 : i] = *reinterpret_cast<const lm_s16x8*>(
            src.v + (kv0 + n0 + key) * src.v_row + hk * src.v_head + d);
    }
  };
  auto stage_write = [&](int buf) {
#pragma unroll
    for (int i = 0; i < KPC; ++i) {
      const int p = tid + i * NW * 64;
      const int key = p / q8, d = (p % q8) * 8;
      if (key < BN)
        *reinterpret_cast<lm_s16x8*>(&lk[buf][key * KP + d]) = kreg[i];
    }
    if (SAME) {
      if (tid < BN) ls[buf][tid] = sreg;
      return;
    }
#pragma unroll
    for (int i = 0; i < VPC; ++i) {
      const int p = tid + i * NW * 64;
      const int key = p / v8, d = (p % v8) * 8;
      if (key < BN)
        *reinterpret_cast<lm_s16x8*>(&lv[buf][key * VPP + d]) =
            vreg[SAME ? 0 : i];
    }
  };

  const int q_first = p0 + wave * 16, q_last = q_first + 15;
  // rows that any query of the tile sees: the first `keep`, then from n_begin
  const int n_begin = window > 0 ? max(pooled, p0 - window + 1 - skip) : 0;
  const int n_end = min(nk, p0 + len - skip);
  // of the pooled rows, those that the tile's last query sees
  const int front =
      pool > 0 ? min(pooled, max(0, p0 + len - window) / pool) : keep;
  auto next_tile = [&](int n0) {
    return n0 + BN >= front ? max(n0 + BN, n_begin) : n0 + BN;
  };
  const int my_q = p0 + qrow;
  const int my_lo = window > 0 ? my_q - window : -1;  // sees keys > my_lo

  auto compute = [&](int n0, int buf) {
    // positions of the tile's rows; it may hold kept rows and others
    const int a0 = place(n0), a1 = place(n0 + BN - 1);
    // pooled rows and tokens in one tile: no order of positions
    const bool both = pool > 0 && n0 < keep && n0 + BN > keep;
    if (!both &&
        (a0 > q_last || (window > 0 && n0 >= keep && a1 <= q_first - window)))
      return;  // nothing of this tile for any query of the wave
    lm_f32x4 s[BN / 16];
#pragma unroll
    for (int t = 0; t < BN / 16; ++t) s[t] = lm_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kc = 0; kc < QS; ++kc) {
      if (kc * 32 < QD) {
#pragma unroll
        for (int t = 0; t < BN / 16; ++t) {
          const lm_s16x8 kf = *reinterpret_cast<const lm_s16x8*>(
              &lk[buf][(t * 16 + r16) * KP + kc * 32 + ko]);
          s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[kc], s[t], 0,
                                                         0, 0);
        }
      }
    }
    const bool full = !both && n0 + BN <= nk && a1 <= q_first &&
                      (window <= 0 || n0 + BN <= keep ||
                       (n0 >= keep && a0 > q_last - window));
    float mx = -INFINITY;
#pragma unroll
    for (int t = 0; t < BN / 16; ++t) {
      if (SAME) {
        const lm_f32x4 ks =
            *reinterpret_cast<const lm_f32x4*>(&ls[buf][16 * t + 4 * g]);
#pragma unroll
        for (int r = 0; r < 4; ++r) s[t][r] *= ks[r];
      }
      if (score.capped) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          s[t][r] = score.out2 * cap_tanh<bf16>(s[t][r] * score.in);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r) s[t][r] *= score.scale2;
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (!full) {
          const int n = n0 + 16 * t + 4 * g + r;
          const int key = place(n);
          const bool see = key <= my_q &&
                           (key > my_lo || (pool > 0 ? n : key) < keep) &&
                           n < nk;
          s[t][r] = see ? s[t][r] : -INFINITY;
        }
        mx = fmaxf(mx, s[t][r]);
      }
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float m_new = fmaxf(m_run, mx);
    // before a query's first visible key m_new is -inf: all weights are 0
    const float m_use = m_new == -INFINITY ? 0.f : m_new;
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_use);
    float sum = 0.f;
#pragma unroll
    for (int t = 0; t < BN / 16; ++t) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        s[t][r] = __builtin_amdgcn_exp2f(s[t][r] - m_use);
        sum += s[t][r];
      }
    }
    l_run = l_run * alpha + sum;
    m_run = m_new;
#pragma unroll
    for (int i = 0; i < VT; ++i) acc[i] *= alpha;
#pragma unroll
    for (int kc = 0; kc < BN / 32; ++kc) {
      const Frag<bf16> pf = frag_of<bf16>(s[2 * kc], s[2 * kc + 1]);
#pragma unroll
      for (int i = 0; i < VT; ++i) {
        if (i * 16 < VP)
          acc[i] = mma32(
              SAME ? load_frag_rows((const bf16*)&lk[buf][kc * 32 * KP +
                                                          i * 16], KP)
                   : load_frag_rows(&lv[buf][kc * 32 * VPP + i * 16], VPP),
              pf, acc[i]);
      }
    }
  };

  int n0 = front > 0 ? 0 : n_begin;
  if (n0 < n_end) {
    stage_load(n0);
    stage_write(0);
  }
  __syncthreads();
  int cur = 0;
  while (n0 < n_end) {
    const int n1 = next_tile(n0);
    const bool more = n1 < n_end;
    if (more) stage_load(n1);
    compute(n0, cur);
    if (more) {
      stage_write(cur ^ 1);
      __syncthreads();
      cur ^= 1;
    }
    n0 = n1;
  }

  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  if (qrow < len) {
    const float sk =
        sink ? __bfloat162float(sink[h]) * LM_LOG2E : -INFINITY;
    const float inv = over_weights(m_run, l_run, sk) * dst_.scale;
    bf16* dst = dst_.out + (t0 + qrow) * dst_.ld + h * VP;
#pragma unroll
    for (int i = 0; i < VT; ++i) {
      if (i * 16 < VP) {
        float f[4] = {acc[i][0] * inv, acc[i][1] * inv, acc[i][2] * inv,
                      acc[i][3] * inv};
        if (dst_.gate) {
          union { uint2 u; bf16 b[4]; } gt;
          gt.u = *reinterpret_cast<const uint2*>(
              dst_.gate + (t0 + qrow) * dst_.ld_gate + h * VP + i * 16 +
              4 * g);
#pragma unroll
          for (int r = 0; r < 4; ++r)
            f[r] *= sigmoid_f(__bfloat162float(gt.b[r]));
        }
        store4(dst + i * 16 + 4 * g, f);
      }
    }
  }
}

void launch_prompt(const torch::Tensor& q, const PromptKeys& src, bool same,
                   const c10::optional<torch::Tensor>& sink,
                   const PromptOut& out, const torch::Tensor& qtiles, int H,
                   int QD, int VP, long window, long keep, long pool,
                   const Score& score) {
  LM_CHECK_I32(qtiles);
  TORCH_CHECK(qtiles.dim() == 2 && qtiles.size(1) == (pool ? 7 : 6));
  TORCH_CHECK(q.scalar_type() == at::kBFloat16 && q.dim() == 2 &&
              q.stride(1) == 1 && q.stride(0) % 8 == 0 &&
              q.size(1) >= (long)H * QD && q.storage_offset() % 8 == 0);
  if (sink) {
    LM_CHECK_CONTIG(*sink);
    TORCH_CHECK(sink->numel() == H && sink->scalar_type() == at::kBFloat16);
  }
  TORCH_CHECK(QD <= 256 && VP <= 256, "prompt attention: head too large");
  TORCH_CHECK(window >= 0 && keep >= 0 && pool >= 0 &&
              ((keep == 0 && pool == 0) || window > 0) &&
              (keep == 0 || pool == 0));
  const int n = qtiles.size(0);
  if (n == 0) return;
  TORCH_CHECK(n <= 65535);
  hipStream_t st = cmls::current_stream();
#define LM_LP(QS, VT, SAME)                                                  \
  hipLaunchKernelGGL((prompt_attn_kernel<QS, VT, SAME>), dim3(H, n),         \
                     dim3(NW * 64), 0, st, (const bf16*)q.data_ptr(),        \
                     q.stride(0), src,                                       \
                     sink ? (const bf16*)sink->data_ptr() : nullptr, out,    \
                     qtiles.data_ptr<int>(), H, QD, VP, (int)window,         \
                     (int)keep, (int)pool, score)
#define LM_LP_V(QS)                                                          \
  do {                                                                       \
    if (VP <= 32) LM_LP(QS, 2, false);                                       \
    else if (VP <= 64) LM_LP(QS, 4, false);                                  \
    else if (VP <= 96) LM_LP(QS, 6, false);                                  \
    else if (VP <= 128) LM_LP(QS, 8, false);                                 \
    else LM_LP(QS, 16, false);                                               \
  } while (0)
  if (same) {
    TORCH_CHECK(QD == VP);
    if (QD <= 32) LM_LP(1, 2, true);
    else if (QD <= 64) LM_LP(2, 4, true);
    else if (QD <= 96) LM_LP(3, 6, true);
    else if (QD <= 128) LM_LP(4, 8, true);
    else LM_LP(8, 16, true);
  } else if (QD <= 64) LM_LP_V(2);
  else if (QD <= 96) LM_LP_V(3);
  else if (QD <= 128) LM_LP_V(4);
  else if (QD <= 192) LM_LP_V(6);
  else LM_LP_V(8);
#undef LM_LP_V
#undef LM_LP
  LM_LAUNCHED();
}

}  // namespace

// q [T, heads * (DP + RP)] (row stride free); kv [rows, H*(DP + VP)] =
// [keys | values]; lat [rows, CP + RP]; gate [T, H * VP] (row stride free);
// out [T, H, VP]: rows of the tiles
void lm_latent_prompt(torch::Tensor q, torch::Tensor kv, torch::Tensor lat,
                      c10::optional<torch::Tensor> sink, torch::Tensor qtiles,
                      torch::Tensor out, long H, long DP, long RP, long CP,
                      long VP, long window, double scale,
                      c10::optional<torch::Tensor> gate) {
  LM_CHECK_CUDA(q);
  LM_CHECK_CONTIG(kv);
  LM_CHECK_CONTIG(lat);
  LM_CHECK_CONTIG(out);
  for (const auto* p : {&kv, &lat, &out})
    TORCH_CHECK(p->scalar_type() == at::kBFloat16,
                "lm_latent_prompt: bf16 only");
  TORCH_CHECK(DP % 32 == 0 && RP % 32 == 0 && CP % 32 == 0 && VP % 32 == 0);
  TORCH_CHECK(kv.dim() == 2 && kv.size(1) == H * (DP + VP));
  TORCH_CHECK(lat.dim() == 2 && lat.size(1) == CP + RP &&
              lat.size(0) == kv.size(0));
  const long T = q.size(0);
  if (gate) lm_check_rows(*gate, T, H * VP, at::kBFloat16);
  TORCH_CHECK(out.size(0) == T && out.numel() == T * H * VP);
  PromptKeys src{};
  src.k = (const bf16*)kv.data_ptr();
  src.v = src.k + H * DP;
  src.rot = (const bf16*)lat.data_ptr() + CP;
  src.k_row = src.v_row = kv.size(1);
  src.rot_row = lat.size(1);
  src.k_head = src.kd = (int)DP;
  src.v_head = (int)VP;
  src.per = 1;
  const PromptOut po{gate ? (const bf16*)gate->data_ptr() : nullptr,
                     gate ? gate->stride(0) : 0L, (bf16*)out.data_ptr(),
                     H * VP, 1.f};
  launch_prompt(q, src, false, sink, po, qtiles, (int)H, (int)(DP + RP),
                (int)VP, window, 0, 0, make_score(scale, 0.0));
}

// q [T, H * KD] (row stride free); rows [n, ROW] gathered cache rows, G slices
// [key KD | value VD], or with `same` [key = value KD] and behind the slices a
// float per head; out [T, H * VD] (row stride free): rows of the tiles
void lm_grouped_prompt(torch::Tensor q, torch::Tensor rows,
                       c10::optional<torch::Tensor> sink,
                       torch::Tensor qtiles, torch::Tensor out, long H, long G,
                       long KD, long VD, bool same, long window, long keep,
                       long pool, double scale, double cap,
                       double out_scale) {
  LM_CHECK_CONTIG(rows);
  TORCH_CHECK(rows.dim() == 2 && rows.scalar_type() == at::kBFloat16 &&
              out.scalar_type() == at::kBFloat16);
  TORCH_CHECK(G >= 1 && H % G == 0 && KD % 32 == 0 && VD % 32 == 0);
  const long SL = same ? KD : KD + VD;
  TORCH_CHECK(rows.size(1) >= G * SL + (same ? 2 * G : 0) &&
              rows.size(1) % 8 == 0);
  lm_check_rows(out, q.size(0), H * VD, at::kBFloat16);
  PromptKeys src{};
  src.k = (const bf16*)rows.data_ptr();
  src.v = src.k + KD;
  src.k_row = src.v_row = rows.size(1);
  src.k_head = src.v_head = (int)SL;
  src.kd = (int)KD;
  src.per = (int)(H / G);
  if (same) {
    src.kscale = (const float*)(src.k + G * SL);
    src.s_row = rows.size(1) / 2;
  }
  const PromptOut po{nullptr, 0L, (bf16*)out.data_ptr(), out.stride(0),
                     (float)out_scale};
  launch_prompt(q, src, same, sink, po, qtiles, (int)H, (int)KD, (int)VD,
                window, keep, pool, make_score(scale, cap));
}
