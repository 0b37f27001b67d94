// Real-gated linear recurrent unit behind a short causal convolution.
//
//   u = conv(x + bx) + bc          r = sigmoid(Ra u + ba), i = sigmoid(Ri u + bi)
//   log a = -8 r softplus(lam)     S = a S + sqrt(1 - a^2) i u
//   out = S * gelu_tanh(y + by)
//
// Ra and Ri are block-diagonal; a workgroup takes one block, so the gate
// products are small dense MFMA tiles on u in LDS and the gates never leave
// registers. Gates, decays and S are float.
//
// Prompts: the recurrence runs over tiles of TT tokens. Pass 1 makes u and
// each tile's composite (prod a, S from zero); pass 2 chains the composites
// per channel and advances the stored state; pass 3 recomputes the gates
// (cheaper than two float arrays through HBM) and replays each tile from its
// carry. Single tokens: one fused kernel, 16 sequences per workgroup.
//
// State per slot: S [W] float, and the last conv inputs as a ring
// [taps][W] indexed by position mod taps, before the bias, so that a
// sequence's first tokens see true zeros. The ring holds one entry more than
// the convolution looks back: a token's own entry is never one that it, or a
// workgroup still working on the same token, reads.
#include "lm_common.h"

namespace {

constexpr int NWV = 4;

__device__ __forceinline__ void decay_and_input(float zr, float zi, float sp,
                                                float u, float* a, float* b) {
  const float la = -8.f * sigmoid_f(zr) * sp;
  const float d = one_minus_exp_f(la);  // 1 - a, exact also for a near 1
  *a = 1.f - d;
  *b = __builtin_amdgcn_sqrtf(d * (2.f - d)) * sigmoid_f(zi) * u;
}

// pre-activations of 16 channels x MT*16 tokens:
// z[mt][r] belongs to token mt*16 + 4*(lane>>4) + r, channel n0 + (lane&15)
template <typename T, int MT>
__device__ __forceinline__ void gate_products(const T* us, int pitch,
                                              const T* ra, const T* ri,
                                              int n0, int BP, lm_f32x4* zr,
                                              lm_f32x4* zi) {
  const int lane = threadIdx.x & 63;
  const int r16 = lane & 15, ko = (lane >> 4) * 8;
  const T* pr = ra + (long)(n0 + r16) * BP + ko;
  const T* pi = ri + (long)(n0 + r16) * BP + ko;
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    zr[m] = lm_f32x4{0.f, 0.f, 0.f, 0.f};
    zi[m] = lm_f32x4{0.f, 0.f, 0.f, 0.f};
  }
#pragma unroll 4
  for (int k = 0; k < BP; k += 32) {
    const Frag<T> wr = load_frag(pr + k), wi = load_frag(pi + k);
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      const Frag<T> uf = load_frag(us + (m * 16 + r16) * pitch + k + ko);
      zr[m] = mma32(uf, wr, zr[m]);
      zi[m] = mma32(uf, wi, zi[m]);
    }
  }
}

// u for 8 channels of one token; xin(d) adds the input d tokens back times
// its tap, already gated on the sequence start
template <typename T>
__device__ __forceinline__ void conv_tap(const T* x, const float* bx,
                                         const T* cw, float* u) {
  float f[8], w[8];
  load8<T>(x, f);
  load8<T>(cw, w);
#pragma unroll
  for (int e = 0; e < 8; ++e) u[e] += (f[e] + bx[e]) * w[e];
}

// tiles: int32 [n, 5] = first token (flat), tokens, first position, state
// slot, distance to the portion's first token
template <typename T, int TT>
__global__ __launch_bounds__(256) void rglru_tile_kernel(
    const T* __restrict__ yx, int ld, const T* __restrict__ byx,
    const T* __restrict__ cw, const T* __restrict__ cb,
    const T* __restrict__ ra, const T* __restrict__ ba,
    const T* __restrict__ ri, const T* __restrict__ bi,
    const T* __restrict__ lam, const T* __restrict__ ring,
    const int* __restrict__ tiles, T* __restrict__ u_out,
    float* __restrict__ comp, int W, int BP, int taps, int n_state) {
  constexpr int MT = TT / 16;
  extern __shared__ __align__(16) char smem[];
  T* us = (T*)smem;
  const int pitch = BP + 8;
  const int tile = blockIdx.x, ch0 = blockIdx.y * BP;
  const int* td = tiles + tile * 5;
  const int t0 = td[0], len = td[1], p0 = td[2], slot = td[3], into = td[4];
  const bool has_state = slot >= 0 && slot < n_state;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int bp8 = BP / 8;
  for (int i = tid; i < TT * bp8; i += 256) {
    const int tt = i / bp8, c = (i % bp8) * 8, ch = ch0 + c;
    float u[8];
    if (tt < len) {
      float bx[8];
      load8<T>(byx + W + ch, bx);
      load8<T>(cb + ch, u);
      for (int d = 0; d < taps; ++d) {
        const int p = p0 + tt - d;
        if (p < 0) break;
        const T* src;
        if (d <= tt + into) {
          src = yx + (long)(t0 + tt - d) * ld + W + ch;
        } else {
          if (!has_state) break;
          src = ring + ((long)slot * taps + p % taps) * W + ch;
        }
        conv_tap<T>(src, bx, cw + (long)(taps - 1 - d) * W + ch, u);
      }
      store8(us + tt * pitch + c, u);
      copy8(u_out + (long)(t0 + tt) * W + ch, us + tt * pitch + c);
    } else {
      zero8(us + tt * pitch + c);
    }
  }
  __syncthreads();
  const long wofs = (long)blockIdx.y * BP * BP;
  const int g = lane >> 4;
  for (int n0 = wave * 16; n0 < BP; n0 += NWV * 16) {
    lm_f32x4 zr[MT], zi[MT];
    gate_products<T, MT>(us, pitch, ra + wofs, ri + wofs, n0, BP, zr, zi);
    const int c = n0 + (lane & 15), ch = ch0 + c;
    const float vr = to_f32(ba[ch]), vi = to_f32(bi[ch]);
    const float sp = softplus_f(to_f32(lam[ch]));
    float A = 1.f, B = 0.f;  // composite of the tile so far
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      float a4 = 1.f, b4 = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int tt = m * 16 + 4 * g + r;
        float a, b;
        decay_and_input(zr[m][r] + vr, zi[m][r] + vi, sp,
                        to_f32(us[tt * pitch + c]), &a, &b);
        if (tt < len) { b4 = a * b4 + b; a4 *= a; }
      }
      // chain the four lane groups, earlier tokens in lower groups
#pragma unroll
      for (int d = 16; d < 64; d <<= 1) {
        const float ap = __shfl_up(a4, d, 64), bp = __shfl_up(b4, d, 64);
        if (lane >= d) { b4 = a4 * bp + b4; a4 *= ap; }
      }
      const float at = __shfl(a4, 48 + (lane & 15), 64);
      const float bt = __shfl(b4, 48 + (lane & 15), 64);
      B = at * B + bt;
      A *= at;
    }
    if (g == 0) {
      float* cp = comp + ((long)tile * 2) * W + ch;
      cp[0] = A;
      cp[W] = B;
    }
  }
}

// per sequence and channel: chain the tiles' composites. comp's first row of
// a tile becomes the state ahead of it. seqs: int32 [n, 6] = first tile,
// tiles, first token, tokens, first position, state slot
template <typename T>
__global__ __launch_bounds__(64) void rglru_carry_kernel(
    float* __restrict__ comp, const int* __restrict__ seqs,
    float* __restrict__ state, T* __restrict__ ring,
    const T* __restrict__ yx, int ld, int W, int taps, int n_state) {
  const int ch = blockIdx.x * 64 + threadIdx.x;
  if (ch >= W) return;
  const int* sd = seqs + blockIdx.y * 6;
  const int tile0 = sd[0], n = sd[1], t0 = sd[2], len = sd[3], p0 = sd[4],
            slot = sd[5];
  const bool has_state = slot >= 0 && slot < n_state;
  float S = (p0 > 0 && has_state) ? state[(long)slot * W + ch] : 0.f;
  float* cp = comp + (long)tile0 * 2 * W + ch;
  int j = 0;
  for (; j + 8 <= n; j += 8) {
    float a[8], b[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      a[e] = cp[(long)(j + e) * 2 * W];
      b[e] = cp[(long)(j + e) * 2 * W + W];
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      cp[(long)(j + e) * 2 * W] = S;
      S = a[e] * S + b[e];
    }
  }
  for (; j < n; ++j) {
    const float a = cp[(long)j * 2 * W], b = cp[(long)j * 2 * W + W];
    cp[(long)j * 2 * W] = S;
    S = a * S + b;
  }
  if (!has_state) return;
  state[(long)slot * W + ch] = S;
  for (int d = min(taps, len) - 1; d >= 0; --d) {
    const int p = p0 + len - 1 - d;
    ring[((long)slot * taps + p % taps) * W + ch] =
        yx[(long)(t0 + len - 1 - d) * ld + W + ch];
  }
}

template <typename T, int TT>
__global__ __launch_bounds__(256) void rglru_out_kernel(
    const T* __restrict__ yx, int ld, const T* __restrict__ byx,
    const T* __restrict__ u_in, const T* __restrict__ ra,
    const T* __restrict__ ba, const T* __restrict__ ri,
    const T* __restrict__ bi, const T* __restrict__ lam,
    const int* __restrict__ tiles, const float* __restrict__ comp,
    T* __restrict__ out, int W, int BP) {
  constexpr int MT = TT / 16;
  extern __shared__ __align__(16) char smem[];
  T* us = (T*)smem;
  const int pitch = BP + 8;
  T* ys = us + TT * pitch;  // y, then the result
  const int tile = blockIdx.x, ch0 = blockIdx.y * BP;
  const int* td = tiles + tile * 5;
  const int t0 = td[0], len = td[1];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int bp8 = BP / 8;
  for (int i = tid; i < TT * bp8; i += 256) {
    const int tt = i / bp8, c = (i % bp8) * 8;
    if (tt < len) {
      copy8(us + tt * pitch + c, u_in + (long)(t0 + tt) * W + ch0 + c);
      copy8(ys + tt * pitch + c, yx + (long)(t0 + tt) * ld + ch0 + c);
    } else {
      zero8(us + tt * pitch + c);
      zero8(ys + tt * pitch + c);
    }
  }
  __syncthreads();
  const long wofs = (long)blockIdx.y * BP * BP;
  const int g = lane >> 4;
  for (int n0 = wave * 16; n0 < BP; n0 += NWV * 16) {
    lm_f32x4 zr[MT], zi[MT];
    gate_products<T, MT>(us, pitch, ra + wofs, ri + wofs, n0, BP, zr, zi);
    const int c = n0 + (lane & 15), ch = ch0 + c;
    const float vr = to_f32(ba[ch]), vi = to_f32(bi[ch]);
    const float sp = softplus_f(to_f32(lam[ch]));
    const float by = to_f32(byx[ch]);
    float S = comp[(long)tile * 2 * W + ch];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      float a[4], b[4];
      float a4 = 1.f, b4 = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int tt = m * 16 + 4 * g + r;
        decay_and_input(zr[m][r] + vr, zi[m][r] + vi, sp,
                        to_f32(us[tt * pitch + c]), &a[r], &b[r]);
        if (tt >= len) { a[r] = 1.f; b[r] = 0.f; }
        b4 = a[r] * b4 + b[r];
        a4 *= a[r];
      }
#pragma unroll
      for (int d = 16; d < 64; d <<= 1) {
        const float ap = __shfl_up(a4, d, 64), bp = __shfl_up(b4, d, 64);
        if (lane >= d) { b4 = a4 * bp + b4; a4 *= ap; }
      }
      // state ahead of this lane's four tokens
      const float ae = __shfl_up(a4, 16, 64), be = __shfl_up(b4, 16, 64);
      float s = g == 0 ? S : ae * S + be;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int tt = m * 16 + 4 * g + r;
        s = a[r] * s + b[r];
        T* yp = ys + tt * pitch + c;  // read and written by this lane only
        *yp = from_f32<T>(s * gelu_tanh_f(to_f32(*yp) + by));
      }
      S = __shfl(a4, 48 + (lane & 15), 64) * S +
          __shfl(b4, 48 + (lane & 15), 64);
    }
  }
  __syncthreads();
  for (int i = tid; i < len * bp8; i += 256) {
    const int tt = i / bp8, c = (i % bp8) * 8;
    copy8(out + (long)(t0 + tt) * W + ch0 + c, ys + tt * pitch + c);
  }
}

// one token each of up to 16 sequences per workgroup; blockIdx.z takes a
// slice of 64 of the block's channels
template <typename T>
__global__ __launch_bounds__(256) void rglru_step_kernel(
    const T* __restrict__ yx, int ld, const T* __restrict__ byx,
    const T* __restrict__ cw, const T* __restrict__ cb,
    const T* __restrict__ ra, const T* __restrict__ ba,
    const T* __restrict__ ri, const T* __restrict__ bi,
    const T* __restrict__ lam, const int* __restrict__ positions,
    const int* __restrict__ slots, float* __restrict__ state,
    T* __restrict__ ring, T* __restrict__ out, int n, int W, int BP,
    int taps, int n_state) {
  extern __shared__ __align__(16) char smem[];
  T* us = (T*)smem;
  const int pitch = BP + 8;
  const int row0 = blockIdx.x * 16, ch0 = blockIdx.y * BP;
  const int s0 = blockIdx.z * 64;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int bp8 = BP / 8;
  // what the second half needs and the first does not change is loaded
  // ahead of it: gate weights, state, gated branch
  const int n0 = s0 + wave * 16;
  const bool active = n0 < BP;
  const int r16 = lane & 15, ko = (lane >> 4) * 8;
  const int c0 = n0 + r16, cch = ch0 + c0;
  constexpr int PK = 4;  // k steps of weights in registers
  Frag<T> wr[PK], wi[PK];
  float s_old[4], y_in[4];
  int slot4[4];
  const T* pr = ra + (long)blockIdx.y * BP * BP + (long)c0 * BP + ko;
  const T* pi = ri + (long)blockIdx.y * BP * BP + (long)c0 * BP + ko;
  if (active) {
#pragma unroll
    for (int k = 0; k < PK; ++k) {
      if (k * 32 < BP) {
        wr[k] = load_frag(pr + k * 32);
        wi[k] = load_frag(pi + k * 32);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = row0 + 4 * (lane >> 4) + r;
      slot4[r] = -1;
      s_old[r] = y_in[r] = 0.f;
      if (t < n) {
        const int slot = slots[t];
        y_in[r] = to_f32(yx[(long)t * ld + cch]);
        if (slot >= 0 && slot < n_state) {
          slot4[r] = slot;
          if (positions[t] > 0) s_old[r] = state[(long)slot * W + cch];
        }
      }
    }
  }
  for (int i = tid; i < 16 * bp8; i += 256) {
    const int rr = i / bp8, c = (i % bp8) * 8, ch = ch0 + c;
    const int t = row0 + rr;
    if (t >= n) {
      zero8(us + rr * pitch + c);
      continue;
    }
    const int pos = positions[t], slot = slots[t];
    const bool has_state = slot >= 0 && slot < n_state;
    float u[8], bx[8];
    load8<T>(byx + W + ch, bx);
    load8<T>(cb + ch, u);
    const T* cur = yx + (long)t * ld + W + ch;
    conv_tap<T>(cur, bx, cw + (long)(taps - 1) * W + ch, u);
    if (has_state) {
#pragma unroll 4
      for (int d = 1; d < min(taps, pos + 1); ++d)
        conv_tap<T>(ring + ((long)slot * taps + (pos - d) % taps) * W + ch,
                    bx, cw + (long)(taps - 1 - d) * W + ch, u);
      // this slice's part of the ring; nobody reads this entry at this step
      if (c >= s0 && c < s0 + 64)
        copy8(ring + ((long)slot * taps + pos % taps) * W + ch, cur);
    }
    store8(us + rr * pitch + c, u);
  }
  __syncthreads();
  if (!active) return;
  lm_f32x4 zr = {0.f, 0.f, 0.f, 0.f}, zi = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int k = 0; k < PK; ++k) {
    if (k * 32 < BP) {
      const Frag<T> uf = load_frag(us + r16 * pitch + k * 32 + ko);
      zr = mma32(uf, wr[k], zr);
      zi = mma32(uf, wi[k], zi);
    }
  }
#pragma unroll 4
  for (int k = PK * 32; k < BP; k += 32) {
    const Frag<T> uf = load_frag(us + r16 * pitch + k + ko);
    zr = mma32(uf, load_frag(pr + k), zr);
    zi = mma32(uf, load_frag(pi + k), zi);
  }
  const float vr = to_f32(ba[cch]), vi = to_f32(bi[cch]);
  const float sp = softplus_f(to_f32(lam[cch]));
  const float by = to_f32(byx[cch]);
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int rr = 4 * (lane >> 4) + r, t = row0 + rr;
    if (t >= n) continue;
    float a, b;
    decay_and_input(zr[r] + vr, zi[r] + vi, sp, to_f32(us[rr * pitch + c0]),
                    &a, &b);
    const float S = a * s_old[r] + b;  // s_old: 0 at position 0
    if (slot4[r] >= 0) state[(long)slot4[r] * W + cch] = S;
    out[(long)t * W + cch] = from_f32<T>(S * gelu_tanh_f(y_in[r] + by));
  }
}

struct RglruDims {
  int T, ld, W, BP, blocks, taps, n_state;
};

RglruDims rglru_check(const torch::Tensor& yx, const torch::Tensor& byx,
                      const torch::Tensor& cw, const torch::Tensor& cb,
                      const torch::Tensor& ra, const torch::Tensor& ba,
                      const torch::Tensor& ri, const torch::Tensor& bi,
                      const torch::Tensor& lam, const torch::Tensor& state,
                      const torch::Tensor& ring) {
  RglruDims d;
  for (const auto* p : {&yx, &byx, &cw, &cb, &ra, &ba, &ri, &bi, &lam, &ring}) {
    TORCH_CHECK(p->is_cuda() && p->is_contiguous() &&
                    p->scalar_type() == yx.scalar_type(),
                "rglru: operands must be contiguous and of one type");
  }
  TORCH_CHECK(ra.dim() == 3 && ra.size(1) == ra.size(2) &&
              ri.sizes() == ra.sizes());
  d.blocks = ra.size(0);
  d.BP = ra.size(1);
  d.W = d.blocks * d.BP;
  d.T = yx.size(0);
  d.ld = yx.size(1);
  d.taps = cw.size(0);
  d.n_state = state.size(0);
  TORCH_CHECK(d.BP % 32 == 0 && d.ld == 2 * d.W && d.taps >= 1);
  TORCH_CHECK(byx.numel() == 2 * d.W && cw.numel() == (long)d.taps * d.W);
  TORCH_CHECK(cb.numel() == d.W && ba.numel() == d.W && bi.numel() == d.W &&
              lam.numel() == d.W);
  TORCH_CHECK(state.is_cuda() && state.is_contiguous() &&
              state.scalar_type() == at::kFloat && state.dim() == 2 &&
              state.size(1) == d.W);
  TORCH_CHECK(ring.dim() == 3 && ring.size(0) == d.n_state &&
              ring.size(1) == d.taps && ring.size(2) == d.W);
  TORCH_CHECK(d.blocks <= 65535);
  return d;
}

template <typename K>
void allow_lds(K fn, int bytes) {
  if (bytes > 64 * 1024)
    HIP_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(fn),
                                  hipFuncAttributeMaxDynamicSharedMemorySize,
                                  bytes));
}

}  // namespace

// rows of `out` that the tiles cover are written; tiles [n, 5], seqs [m, 6]
// of `tile` tokens at most
void lm_rglru_prefill(torch::Tensor yx, torch::Tensor byx, torch::Tensor cw,
                      torch::Tensor cb, torch::Tensor ra, torch::Tensor ba,
                      torch::Tensor ri, torch::Tensor bi, torch::Tensor lam,
                      torch::Tensor state, torch::Tensor ring,
                      torch::Tensor tiles, torch::Tensor seqs,
                      torch::Tensor out, long tile) {
  const RglruDims d =
      rglru_check(yx, byx, cw, cb, ra, ba, ri, bi, lam, state, ring);
  LM_CHECK_I32(tiles);
  LM_CHECK_I32(seqs);
  LM_CHECK_CONTIG(out);
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 5);
  TORCH_CHECK(seqs.dim() == 2 && seqs.size(1) == 6);
  TORCH_CHECK(out.size(0) == d.T && out.size(1) == d.W &&
              out.scalar_type() == yx.scalar_type());
  TORCH_CHECK(tile == 64 || tile == 16, "rglru: tile is 64 or 16 tokens");
  const int nt = tiles.size(0), ns = seqs.size(0);
  if (nt == 0) return;
  TORCH_CHECK(ns <= 65535);
  const int bytes = (int)(tile * (d.BP + 8) * yx.element_size());
  TORCH_CHECK(2 * bytes <= 160 * 1024, "rglru: block of ", d.BP,
              " channels does not fit LDS");
  auto u = torch::empty({d.T, d.W}, yx.options());
  auto comp = torch::empty({nt, 2, d.W}, yx.options().dtype(at::kFloat));
  hipStream_t st = cmls::current_stream();
#define P(X) ((const scalar_t*)(X).data_ptr())
#define LM_RG(TT)                                                            \
  do {                                                                       \
    allow_lds(&rglru_tile_kernel<scalar_t, TT>, bytes);                      \
    allow_lds(&rglru_out_kernel<scalar_t, TT>, 2 * bytes);                   \
    hipLaunchKernelGGL((rglru_tile_kernel<scalar_t, TT>), dim3(nt, d.blocks),\
                       dim3(256), bytes, st, P(yx), d.ld, P(byx), P(cw),     \
                       P(cb), P(ra), P(ba), P(ri), P(bi), P(lam), P(ring),   \
                       tiles.data_ptr<int>(), (scalar_t*)u.data_ptr(),       \
                       comp.data_ptr<float>(), d.W, d.BP, d.taps,            \
                       d.n_state);                                           \
    hipLaunchKernelGGL((rglru_carry_kernel<scalar_t>),                       \
                       dim3((d.W + 63) / 64, ns), dim3(64), 0, st,           \
                       comp.data_ptr<float>(), seqs.data_ptr<int>(),         \
                       state.data_ptr<float>(), (scalar_t*)ring.data_ptr(),  \
                       P(yx), d.ld, d.W, d.taps, d.n_state);                 \
    hipLaunchKernelGGL((rglru_out_kernel<scalar_t, TT>), dim3(nt, d.blocks), \
                       dim3(256), 2 * bytes, st, P(yx), d.ld, P(byx), P(u),  \
                       P(ra), P(ba), P(ri), P(bi), P(lam),                   \
                       tiles.data_ptr<int>(), comp.data_ptr<float>(),        \
                       (scalar_t*)out.data_ptr(), d.W, d.BP);                \
  } while (0)
  LM_DISPATCH(yx, "lm_rglru_prefill", [&] {
    if (tile == 64) LM_RG(64);
    else LM_RG(16);
  });
#undef LM_RG
#undef P
  LM_LAUNCHED();
}

// the first n rows: one token of n different sequences
void lm_rglru_step(torch::Tensor yx, torch::Tensor byx, torch::Tensor cw,
                   torch::Tensor cb, torch::Tensor ra, torch::Tensor ba,
                   torch::Tensor ri, torch::Tensor bi, torch::Tensor lam,
                   torch::Tensor state, torch::Tensor ring,
                   torch::Tensor positions, torch::Tensor slots,
                   torch::Tensor out, long n) {
  const RglruDims d =
      rglru_check(yx, byx, cw, cb, ra, ba, ri, bi, lam, state, ring);
  LM_CHECK_I32(positions);
  LM_CHECK_I32(slots);
  LM_CHECK_CONTIG(out);
  TORCH_CHECK(n >= 0 && n <= d.T && positions.numel() >= n &&
              slots.numel() >= n);
  TORCH_CHECK(out.size(0) == d.T && out.size(1) == d.W &&
              out.scalar_type() == yx.scalar_type());
  if (n == 0) return;
  const int bytes = (int)(16 * (d.BP + 8) * yx.element_size());
  TORCH_CHECK(bytes <= 160 * 1024, "rglru: block of ", d.BP,
              " channels does not fit LDS");
#define P(X) ((const scalar_t*)(X).data_ptr())
  LM_DISPATCH(yx, "lm_rglru_step", [&] {
    allow_lds(&rglru_step_kernel<scalar_t>, bytes);
    hipLaunchKernelGGL((rglru_step_kernel<scalar_t>),
                       dim3((n + 15) / 16, d.blocks, (d.BP + 63) / 64),
                       dim3(256), bytes, cmls::current_stream(), P(yx), d.ld,
                       P(byx), P(cw), P(cb), P(ra), P(ba), P(ri), P(bi),
                       P(lam), positions.data_ptr<int>(),
                       slots.data_ptr<int>(), state.data_ptr<float>(),
                       (scalar_t*)ring.data_ptr(), (scalar_t*)out.data_ptr(),
                       (int)n, d.W, d.BP, d.taps, d.n_state);
  });
#undef P
  LM_LAUNCHED();
}
