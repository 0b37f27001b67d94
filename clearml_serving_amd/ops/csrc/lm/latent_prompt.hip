// Latent attention for prompt portions, expanded form: flash attention on
// keys and values that were rebuilt per head from the cached latents.
//
// Per head a key is [nope part | rotated part]; the rotated part is shared by
// all heads and read from the gathered cache rows. The workgroup takes 128
// queries of one head (8 waves x 16) and walks the 64-key tiles that any of
// them can see. S^T = K Q^T leaves each lane with keys of ONE query, so max,
// sum and the running state are lane-local up to two shuffles; and because
// the k order of an MFMA is free, V is read (transposing LDS reads) in the key
// order that the S^T registers already have -- the weights go from registers
// straight into the second product.
#include "lm_common.h"

namespace {

constexpr float LOG2E = 1.4426950408889634f;
constexpr int BM = 128, BN = 64, NW = 8;

// qtiles: int32 [n, 6] = first token (flat), tokens, first position, first
// row in the gathered keys, that row's position, gathered rows
// two workgroups per CU (128 registers) where their LDS fits
template <int QS, int VT>
__global__ __launch_bounds__(NW * 64, QS * 2 + VT <= 16 ? 4 : 2)
void latent_prompt_kernel(
    const bf16* __restrict__ q, long q_t,   // q[t * q_t + h * QD]
    const bf16* __restrict__ kv, int ldkv,  // [rows, H*DP + H*VP]
    const bf16* __restrict__ rot, int ld_rot, const bf16* __restrict__ sink,
    const bf16* __restrict__ gate, long ld_gate,  // [t, H*VP], null: none
    const int* __restrict__ qtiles, bf16* __restrict__ out, int H, int DP,
    int RP, int VP, int window, float scale) {
  constexpr int KP = QS * 32 + 8;   // LDS pitches
  constexpr int VPP = VT * 16 + 8;
  __shared__ __align__(16) short lk[2][BN * KP];
  __shared__ __align__(16) bf16 lv[2][BN * VPP];
  const int QD = DP + RP;
  const int h = blockIdx.x;
  const int* td = qtiles + (long)blockIdx.y * 6;
  const int t0 = td[0], len = td[1], p0 = td[2], kv0 = td[3], k_lo = td[4],
            nk = td[5];
  const int tid = threadIdx.x, lane = tid & 63, wave = uniform_wave();
  const int r16 = lane & 15, g = lane >> 4, ko = g * 8;
  const int qrow = wave * 16 + r16;
  const float scale2 = scale * LOG2E;

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
  lm_s16x8 kreg[KPC], vreg[VPC];
  auto stage_load = [&](int n0) {
#pragma unroll
    for (int i = 0; i < KPC; ++i) {
      const int p = tid + i * NW * 64;
      const int key = p / q8, d = (p % q8) * 8;
      kreg[i] = lm_s16x8{0, 0, 0, 0, 0, 0, 0, 0};
      if (key < BN && n0 + key < nk) {
        const long row = kv0 + n0 + key;
        kreg[i] = *reinterpret_cast<const lm_s16x8*>(
            d < DP ? kv + row * ldkv + h * DP + d
                   : rot + row * ld_rot + (d - DP));
      }
    }
#pragma unroll
    for (int i = 0; i < VPC; ++i) {
      const int p = tid + i * NW * 64;
      const int key = p / v8, d = (p % v8) * 8;
      vreg[i] = lm_s16x8{0, 0, 0, 0, 0, 0, 0, 0};
      if (key < BN && n0 + key < nk)
        vreg[i] = *reinterpret_cast<const lm_s16x8*>(
            kv + (long)(kv0 + n0 + key) * ldkv + H * DP + h * VP + d);
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
#pragma unroll
    for (int i = 0; i < VPC; ++i) {
      const int p = tid + i * NW * 64;
      const int key = p / v8, d = (p % v8) * 8;
      if (key < BN)
        *reinterpret_cast<lm_s16x8*>(&lv[buf][key * VPP + d]) = vreg[i];
    }
  };

  const int q_first = p0 + wave * 16, q_last = q_first + 15;
  const int n_begin = window > 0 ? max(0, p0 - window + 1 - k_lo) : 0;
  const int n_end = min(nk, p0 + len - k_lo);
  const int my_q = p0 + qrow;
  const int my_lo = window > 0 ? my_q - window : -1;  // sees keys > my_lo

  auto compute = [&](int n0, int buf) {
    const int a0 = k_lo + n0;
    if (a0 > q_last || (window > 0 && a0 + BN - 1 <= q_first - window))
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
    const bool full = n0 + BN <= nk && a0 + BN - 1 <= q_first &&
                      (window <= 0 || a0 > q_last - window);
    float mx = -INFINITY;
#pragma unroll
    for (int t = 0; t < BN / 16; ++t) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float v = s[t][r] * scale2;
        if (!full) {
          const int key = a0 + 16 * t + 4 * g + r;
          v = (key <= my_q && key > my_lo && key < k_lo + nk) ? v : -INFINITY;
        }
        s[t][r] = v;
        mx = fmaxf(mx, v);
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
              load_frag_rows(&lv[buf][kc * 32 * VPP + i * 16], VPP), pf,
              acc[i]);
      }
    }
  };

  if (n_begin < n_end) {
    stage_load(n_begin);
    stage_write(0);
  }
  __syncthreads();
  int cur = 0;
  for (int n0 = n_begin; n0 < n_end; n0 += BN) {
    const bool more = n0 + BN < n_end;
    if (more) stage_load(n0 + BN);
    compute(n0, cur);
    if (more) {
      stage_write(cur ^ 1);
      __syncthreads();
      cur ^= 1;
    }
  }

  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  if (qrow < len) {
    const float sk = sink ? __bfloat162float(sink[h]) * LOG2E : -INFINITY;
    const float m_f = fmaxf(m_run, sk);
    const float e = exp2f(m_run - m_f);
    const float inv = e / (l_run * e + exp2f(sk - m_f));
    bf16* dst = out + ((long)(t0 + qrow) * H + h) * VP;
#pragma unroll
    for (int i = 0; i < VT; ++i) {
      if (i * 16 < VP) {
        float f[4] = {acc[i][0] * inv, acc[i][1] * inv, acc[i][2] * inv,
                      acc[i][3] * inv};
        if (gate) {
          union { uint2 u; bf16 b[4]; } gt;
          gt.u = *reinterpret_cast<const uint2*>(
              gate + (long)(t0 + qrow) * ld_gate + h * VP + i * 16 + 4 * g);
#pragma unroll
          for (int r = 0; r < 4; ++r)
            f[r] *= sigmoid_f(__bfloat162float(gt.b[r]));
        }
        store4(dst + i * 16 + 4 * g, f);
      }
    }
  }
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
  LM_CHECK_I32(qtiles);
  for (const auto* p : {&q, &kv, &lat, &out})
    TORCH_CHECK(p->scalar_type() == at::kBFloat16,
                "lm_latent_prompt: bf16 only");
  const int QD = DP + RP;
  TORCH_CHECK(DP % 32 == 0 && RP % 32 == 0 && CP % 32 == 0 && VP % 32 == 0);
  TORCH_CHECK(q.dim() == 2 && q.stride(1) == 1 && q.stride(0) % 8 == 0 &&
              q.size(1) >= H * QD && q.storage_offset() % 8 == 0);
  TORCH_CHECK(kv.dim() == 2 && kv.size(1) == H * (DP + VP));
  TORCH_CHECK(lat.dim() == 2 && lat.size(1) == CP + RP &&
              lat.size(0) == kv.size(0));
  if (sink) {
    LM_CHECK_CONTIG(*sink);
    TORCH_CHECK(sink->numel() == H && sink->scalar_type() == at::kBFloat16);
  }
  if (gate)
    TORCH_CHECK(gate->is_cuda() && gate->scalar_type() == at::kBFloat16 &&
                gate->dim() == 2 && gate->size(0) == q.size(0) &&
                gate->size(1) == H * VP && gate->stride(1) == 1 &&
                gate->stride(0) % 8 == 0 && gate->storage_offset() % 8 == 0);
  TORCH_CHECK(out.size(0) == q.size(0) && out.numel() == q.size(0) * H * VP);
  TORCH_CHECK(qtiles.dim() == 2 && qtiles.size(1) == 6);
  TORCH_CHECK(QD <= 256 && VP <= 256, "lm_latent_prompt: head too large");
  const int n = qtiles.size(0);
  if (n == 0) return;
  TORCH_CHECK(n <= 65535);
  hipStream_t st = cmls::current_stream();
#define LM_LP(QS, VT)                                                        \
  hipLaunchKernelGGL((latent_prompt_kernel<QS, VT>), dim3(H, n),             \
                     dim3(NW * 64), 0, st, (const bf16*)q.data_ptr(),        \
                     q.stride(0), (const bf16*)kv.data_ptr(),                \
                     (int)kv.size(1), (const bf16*)lat.data_ptr() + CP,      \
                     (int)lat.size(1),                                       \
                     sink ? (const bf16*)sink->data_ptr() : nullptr,         \
                     gate ? (const bf16*)gate->data_ptr() : nullptr,         \
                     gate ? gate->stride(0) : 0L,                            \
                     qtiles.data_ptr<int>(), (bf16*)out.data_ptr(), (int)H,  \
                     (int)DP, (int)RP, (int)VP, (int)window, (float)scale)
#define LM_LP_V(QS)                                                          \
  do {                                                                       \
    if (VP <= 32) LM_LP(QS, 2);                                              \
    else if (VP <= 64) LM_LP(QS, 4);                                         \
    else if (VP <= 96) LM_LP(QS, 6);                                         \
    else if (VP <= 128) LM_LP(QS, 8);                                        \
    else LM_LP(QS, 16);                                                      \
  } while (0)
  if (QD <= 64) LM_LP_V(2);
  else if (QD <= 96) LM_LP_V(3);
  else if (QD <= 128) LM_LP_V(4);
  else if (QD <= 192) LM_LP_V(6);
  else LM_LP_V(8);
#undef LM_LP_V
#undef LM_LP
  LM_LAUNCHED();
}
