// Hyper-connections: the residual is `S` float streams per token. A sublayer
// reads a weighted sum of them, its output goes back to all:
//
//   u = sum_s in[s] X_s,   h = norm(u)
//   X_t <- sum_s mix[s, t] X_s + out[t] y
//
// One kernel does a sublayer's second line and the next one's first, so the
// streams make one round trip to HBM per sublayer. Also the embedding that
// starts them and the cap on the logits.
//
// Coefficients are floats: mix [S][S] (from, to), out [S], the next sublayer's
// in [S] and the gain of its norm, one number for all coordinates.
#include "lm_common.h"

namespace {

constexpr int MAX_S = 8;

// h = u / rms(u) * gain for the row whose u lies in LDS
template <typename T>
__device__ __forceinline__ void norm_row(const float* u, float ss, float gain,
                                         T* __restrict__ h, int width, int n,
                                         float eps, float* tmp) {
  ss = block_reduce(ss, tmp, SumOp{}, 0.f);
  const float f = gain / sqrtf(ss / (float)n + eps);
  for (int c = threadIdx.x * 4; c < width; c += blockDim.x * 4) {
    const lm_f32x4 v = *reinterpret_cast<const lm_f32x4*>(u + c);
    const float o[4] = {v[0] * f, v[1] * f, v[2] * f, v[3] * f};
    store4(h + c, o);
  }
}

__device__ __forceinline__ lm_f32x4 load4f(const float* p) {
  return *reinterpret_cast<const lm_f32x4*>(p);
}
__device__ __forceinline__ lm_f32x4 load4f(const bf16* p) {
  union { uint2 u; bf16 b[4]; } c;
  c.u = *reinterpret_cast<const uint2*>(p);
  return lm_f32x4{to_f32(c.b[0]), to_f32(c.b[1]), to_f32(c.b[2]),
                  to_f32(c.b[3])};
}

// X [T, S, width]; coef: in [S], gain
template <typename T>
__global__ __launch_bounds__(256) void hyper_embed_kernel(
    const long* __restrict__ tokens, const T* __restrict__ table,
    const float* __restrict__ coef, float* __restrict__ x, T* __restrict__ h,
    int S, int width, int n, float eps, long vocab) {
  extern __shared__ __align__(16) float u[];
  __shared__ float tmp[16];
  const long t = blockIdx.x;
  long id = tokens[t];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  float ss = 0.f;
  for (int c = threadIdx.x * 4; c < width; c += blockDim.x * 4) {
    const lm_f32x4 v = load4f(table + id * width + c);
    lm_f32x4 sum = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < S; ++s) {
      *reinterpret_cast<lm_f32x4*>(x + (t * S + s) * width + c) = v;
      sum += coef[s] * v;
    }
    *reinterpret_cast<lm_f32x4*>(u + c) = sum;
    ss += sum[0] * sum[0] + sum[1] * sum[1] + sum[2] * sum[2] +
          sum[3] * sum[3];
  }
  norm_row(u, ss, coef[S], h + t * width, width, n, eps, tmp);
}

// y = o[t], or MIX: the sum over a token's `slots` slots of share * o[pos],
// a slot without a row (pos < 0) stands for `skip`, the sublayer's own input.
// LAST: nobody reads the streams again.
template <typename T, int S, bool MIX, bool LAST>
__global__ __launch_bounds__(256) void hyper_step_kernel(
    const T* __restrict__ o, const int* __restrict__ pos,
    const float* __restrict__ share, int slots, int n_rows,
    const T* __restrict__ skip, const float* __restrict__ coef,
    float* __restrict__ x, T* __restrict__ h, int width, int n, float eps) {
  extern __shared__ __align__(16) float u[];
  __shared__ float tmp[16];
  const long t = blockIdx.x;
  float mix[S][S], out[S], in[S];
#pragma unroll
  for (int a = 0; a < S; ++a) {
#pragma unroll
    for (int b = 0; b < S; ++b) mix[a][b] = coef[a * S + b];
    out[a] = coef[S * S + a];
    in[a] = coef[S * S + S + a];
  }
  float own = 0.f;  // weight of `skip`
  if (MIX && skip)
    for (int k = 0; k < slots; ++k)
      own += pos[t * slots + k] < 0 ? share[t * slots + k] : 0.f;
  float ss = 0.f;
  for (int c = threadIdx.x * 4; c < width; c += blockDim.x * 4) {
    lm_f32x4 v[S];
#pragma unroll
    for (int s = 0; s < S; ++s) v[s] = load4f(x + (t * S + s) * width + c);
    lm_f32x4 y;
    if (MIX) {
      y = lm_f32x4{0.f, 0.f, 0.f, 0.f};
      if (skip) y = own * load4f(skip + t * width + c);
#pragma unroll 4
      for (int k = 0; k < slots; ++k) {
        const long p = pos[t * slots + k];
        if (p >= 0 && p < n_rows)
          y += share[t * slots + k] * load4f(o + p * width + c);
      }
    } else {
      y = load4f(o + t * width + c);
    }
    lm_f32x4 sum = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int b = 0; b < S; ++b) {
      lm_f32x4 w = out[b] * y;
#pragma unroll
      for (int a = 0; a < S; ++a) w += mix[a][b] * v[a];
      if (!LAST)
        *reinterpret_cast<lm_f32x4*>(x + (t * S + b) * width + c) = w;
      sum += in[b] * w;
    }
    *reinterpret_cast<lm_f32x4*>(u + c) = sum;
    ss += sum[0] * sum[0] + sum[1] * sum[1] + sum[2] * sum[2] +
          sum[3] * sum[3];
  }
  norm_row(u, ss, coef[S * S + 2 * S], h + t * width, width, n, eps, tmp);
}

// out[r][c] = cap * tanh(z[r][c] / cap), the first n columns
template <typename T>
__global__ __launch_bounds__(256) void soft_cap_kernel(
    const T* __restrict__ z, float* __restrict__ out, int ld, int n,
    float cap) {
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= n) return;
  const long r = blockIdx.x;
  out[r * n + c] = cap * tanhf(to_f32(z[r * ld + c]) / cap);
}

int threads_for(long width) {
  return width <= 256 ? 64 : width <= 512 ? 128 : 256;
}

void check_coef(const torch::Tensor& c, long n) {
  TORCH_CHECK(c.is_cuda() && c.is_contiguous() && c.numel() == n &&
                  c.scalar_type() == at::kFloat,
              "hyper: coefficients");
}

}  // namespace

// -> {streams float [T, S, width], h [T, width]}; coef: in [S], gain
std::vector<torch::Tensor> lm_hyper_embed(torch::Tensor tokens,
                                          torch::Tensor table,
                                          torch::Tensor coef, long S, long n,
                                          double eps) {
  LM_CHECK_CONTIG(tokens);
  LM_CHECK_CONTIG(table);
  TORCH_CHECK(tokens.scalar_type() == at::kLong && tokens.dim() == 1);
  const int T = tokens.size(0), width = table.size(1);
  TORCH_CHECK(width % 8 == 0 && width <= 16384 && n >= 1 && n <= width);
  TORCH_CHECK(S >= 1 && S <= MAX_S, "hyper: 1 to 8 streams");
  check_coef(coef, S + 1);
  auto x = torch::empty({T, S, width}, table.options().dtype(at::kFloat));
  auto h = torch::empty({T, width}, table.options());
  if (T == 0) return {x, h};
  LM_DISPATCH(table, "lm_hyper_embed", [&] {
    hipLaunchKernelGGL((hyper_embed_kernel<scalar_t>), dim3(T),
                       dim3(threads_for(width)), width * 4,
                       cmls::current_stream(), tokens.data_ptr<long>(),
                       (const scalar_t*)table.data_ptr(),
                       coef.data_ptr<float>(), x.data_ptr<float>(),
                       (scalar_t*)h.data_ptr(), (int)S, width, (int)n,
                       (float)eps, (long)table.size(0));
  });
  LM_LAUNCHED();
  return {x, h};
}

// o: [T, width], or with pos, share [T, slots] the rows they pick and weigh;
// coef: mix [S, S], out [S], in [S], gain. -> h
torch::Tensor lm_hyper_step(torch::Tensor o, torch::Tensor x,
                            torch::Tensor coef, long n, double eps, bool last,
                            c10::optional<torch::Tensor> pos,
                            c10::optional<torch::Tensor> share,
                            c10::optional<torch::Tensor> skip) {
  LM_CHECK_CONTIG(o);
  LM_CHECK_CONTIG(x);
  TORCH_CHECK(o.dim() == 2 && x.dim() == 3 && x.scalar_type() == at::kFloat);
  const int T = x.size(0), S = x.size(1), width = x.size(2);
  TORCH_CHECK(S >= 1 && S <= MAX_S, "hyper: 1 to 8 streams");
  TORCH_CHECK(o.size(1) == width && width % 8 == 0 && width <= 16384);
  TORCH_CHECK(n >= 1 && n <= width);
  check_coef(coef, S * S + 2 * S + 1);
  int slots = 0;
  if (pos) {
    TORCH_CHECK(share.has_value());
    LM_CHECK_I32(*pos);
    LM_CHECK_CONTIG(*share);
    TORCH_CHECK(pos->dim() == 2 && pos->size(0) == T &&
                share->sizes() == pos->sizes() &&
                share->scalar_type() == at::kFloat);
    slots = pos->size(1);
  } else {
    TORCH_CHECK(o.size(0) == T);
  }
  if (skip) {
    LM_CHECK_CONTIG(*skip);
    TORCH_CHECK(pos.has_value() && skip->dim() == 2 && skip->size(0) == T &&
                skip->size(1) == width &&
                skip->scalar_type() == o.scalar_type());
  }
  auto h = torch::empty({T, width}, o.options());
  if (T == 0) return h;
#define LM_HS_(S, MIX, LAST)                                                 \
  hipLaunchKernelGGL((hyper_step_kernel<scalar_t, S, MIX, LAST>), dim3(T),   \
                     dim3(threads_for(width)), width * 4,                    \
                     cmls::current_stream(), (const scalar_t*)o.data_ptr(),  \
                     pos ? pos->data_ptr<int>() : nullptr,                   \
                     share ? share->data_ptr<float>() : nullptr, slots,      \
                     (int)o.size(0),                                         \
                     skip ? (const scalar_t*)skip->data_ptr() : nullptr,     \
                     coef.data_ptr<float>(), x.data_ptr<float>(),            \
                     (scalar_t*)h.data_ptr(), width, (int)n, (float)eps)
#define LM_HS(S)                                                             \
  case S:                                                                    \
    if (pos) {                                                               \
      if (last) LM_HS_(S, true, true); else LM_HS_(S, true, false);          \
    } else {                                                                 \
      if (last) LM_HS_(S, false, true); else LM_HS_(S, false, false);        \
    }                                                                        \
    break
  LM_DISPATCH(o, "lm_hyper_step", [&] {
    switch (S) {
      LM_HS(1); LM_HS(2); LM_HS(3); LM_HS(4);
      LM_HS(5); LM_HS(6); LM_HS(7); LM_HS(8);
    }
  });
#undef LM_HS
#undef LM_HS_
  LM_LAUNCHED();
  return h;
}

// z [R, ld] -> float [R, n]
torch::Tensor lm_soft_cap(torch::Tensor z, long n, double cap) {
  LM_CHECK_CONTIG(z);
  TORCH_CHECK(z.dim() == 2 && n >= 1 && n <= z.size(1) && cap > 0.0);
  const int R = z.size(0);
  auto out = torch::empty({R, n}, z.options().dtype(at::kFloat));
  if (R == 0) return out;
  TORCH_CHECK((n + 255) / 256 <= 65535);
  LM_DISPATCH(z, "lm_soft_cap", [&] {
    hipLaunchKernelGGL((soft_cap_kernel<scalar_t>),
                       dim3(R, (n + 255) / 256), dim3(256), 0,
                       cmls::current_stream(), (const scalar_t*)z.data_ptr(),
                       out.data_ptr<float>(), (int)z.size(1), (int)n,
                       (float)cap);
  });
  LM_LAUNCHED();
  return out;
}
