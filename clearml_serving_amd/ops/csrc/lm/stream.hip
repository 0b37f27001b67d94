// Residual-stream kernels: embedding, norm-on-output with residual add,
// output norm, gated GELU.
//
// The residual x is float; each step that changes it also writes the copy in
// the matrix-product type that the next projection reads, so x makes one
// round trip to HBM per sublayer.
#include "lm_common.h"

namespace {

template <typename T>
__global__ __launch_bounds__(256) void embed_kernel(
    const long* __restrict__ tokens, const T* __restrict__ table,
    float* __restrict__ x, T* __restrict__ h, int width, long vocab) {
  const long t = blockIdx.x;
  long id = tokens[t];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  for (int c = threadIdx.x * 8; c < width; c += 256 * 8) {
    float f[8];
    load8<T>(table + id * width + c, f);
    store8(x + t * width + c, f);
    if (h) store8(h + t * width + c, f);
  }
}

// x += (o + bias) / rms(o + bias) * (1 + w); h = x. Rows of `width`
// (padded) elements of which `n` count; the pad is zero in o, bias and w.
// NV: 8-element vectors a thread keeps in registers.
template <typename T, int NV>
__global__ __launch_bounds__(256) void post_norm_add_kernel(
    const T* __restrict__ o, const T* __restrict__ bias,
    const T* __restrict__ w, float* __restrict__ x, T* __restrict__ h,
    int width, int n, float eps) {
  __shared__ float tmp[16];
  const long row = (long)blockIdx.x * width;
  float v[NV][8];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + threadIdx.x) * 8;
    if (c < width) {
      load8<T>(o + row + c, v[i]);
      if (bias) {
        float b[8];
        load8<T>(bias + c, b);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[i][e] += b[e];
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += v[i][e] * v[i][e];
    }
  }
  ss = block_reduce(ss, tmp, SumOp{}, 0.f);
  const float inv = 1.f / sqrtf(ss / (float)n + eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + threadIdx.x) * 8;
    if (c < width) {
      float g[8], r[8];
      load8<T>(w + c, g);
      load8<float>(x + row + c, r);
#pragma unroll
      for (int e = 0; e < 8; ++e) r[e] += v[i][e] * inv * (1.f + g[e]);
      store8(x + row + c, r);
      if (h) store8(h + row + c, r);
    }
  }
}

// out[i] = norm(x[rows[i]]) * (1 + w) * scale
template <typename T>
__global__ __launch_bounds__(256) void output_norm_kernel(
    const float* __restrict__ x, const int* __restrict__ rows,
    const T* __restrict__ w, T* __restrict__ out, int width, int n,
    int n_tok, float eps, float scale) {
  __shared__ float tmp[16];
  int r = rows ? rows[blockIdx.x] : (int)blockIdx.x;
  r = min(max(r, 0), n_tok - 1);
  const float* src = x + (long)r * width;
  float ss = 0.f;
  for (int c = threadIdx.x * 8; c < width; c += 256 * 8) {
    float f[8];
    load8<float>(src + c, f);
#pragma unroll
    for (int e = 0; e < 8; ++e) ss += f[e] * f[e];
  }
  ss = block_reduce(ss, tmp, SumOp{}, 0.f);
  const float inv = 1.f / sqrtf(ss / (float)n + eps);
  for (int c = threadIdx.x * 8; c < width; c += 256 * 8) {
    float f[8], g[8];
    load8<float>(src + c, f);
    load8<T>(w + c, g);
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] = f[e] * inv * (1.f + g[e]) * scale;
    store8(out + (long)blockIdx.x * width + c, f);
  }
}

// gu = [gate | up] rows of 2*ff; out = gelu_tanh(gate + bg) * (up + bu)
template <typename T>
__global__ __launch_bounds__(256) void gelu_mul_kernel(
    const T* __restrict__ gu, const T* __restrict__ bias,
    T* __restrict__ out, int ff) {
  const long t = blockIdx.x;
  const int c = (blockIdx.y * 256 + threadIdx.x) * 8;
  if (c >= ff) return;
  float g[8], u[8];
  load8<T>(gu + t * 2 * ff + c, g);
  load8<T>(gu + t * 2 * ff + ff + c, u);
  if (bias) {
    float bg[8], bu[8];
    load8<T>(bias + c, bg);
    load8<T>(bias + ff + c, bu);
#pragma unroll
    for (int e = 0; e < 8; ++e) { g[e] += bg[e]; u[e] += bu[e]; }
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) g[e] = gelu_tanh_f(g[e]) * u[e];
  store8(out + t * ff + c, g);
}

// out[i] = src[idx[i]], rows of `width` elements
template <typename T>
__global__ __launch_bounds__(256) void gather_rows_kernel(
    const T* __restrict__ src, const int* __restrict__ idx,
    T* __restrict__ out, int n, int width, long n_src) {
  const int per = width / 8;
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= (long)n * per) return;
  const long r = i / per;
  const int c = (int)(i % per) * 8;
  long s = idx[r];
  s = s < 0 ? 0 : (s >= n_src ? n_src - 1 : s);
  copy8(out + r * width + c, src + s * width + c);
}

}  // namespace

std::vector<torch::Tensor> lm_embed(torch::Tensor tokens,
                                    torch::Tensor table) {
  LM_CHECK_CONTIG(tokens);
  LM_CHECK_CONTIG(table);
  TORCH_CHECK(tokens.scalar_type() == at::kLong && tokens.dim() == 1);
  const int T = tokens.size(0), width = table.size(1);
  TORCH_CHECK(width % 8 == 0, "lm_embed: width % 8");
  auto x = torch::empty({T, width}, table.options().dtype(at::kFloat));
  // in 32-bit runs the stream itself is the projection input
  auto h = table.scalar_type() == at::kFloat ? x : torch::empty(
      {T, width}, table.options());
  if (T == 0) return {x, h};
  LM_DISPATCH(table, "lm_embed", [&] {
    scalar_t* hp = h.data_ptr() == x.data_ptr() ? nullptr
                                                : (scalar_t*)h.data_ptr();
    hipLaunchKernelGGL((embed_kernel<scalar_t>), dim3(T), dim3(256), 0,
                       cmls::current_stream(), tokens.data_ptr<long>(),
                       (const scalar_t*)table.data_ptr(),
                       x.data_ptr<float>(), hp, width, (long)table.size(0));
  });
  LM_LAUNCHED();
  return {x, h};
}

torch::Tensor lm_post_norm_add(torch::Tensor o,
                               c10::optional<torch::Tensor> bias,
                               torch::Tensor w, torch::Tensor x, long n,
                               double eps) {
  LM_CHECK_CONTIG(o);
  LM_CHECK_CONTIG(w);
  LM_CHECK_CONTIG(x);
  const int T = o.size(0), width = o.size(1);
  TORCH_CHECK(x.scalar_type() == at::kFloat && x.sizes() == o.sizes());
  TORCH_CHECK(w.numel() == width && w.scalar_type() == o.scalar_type());
  TORCH_CHECK(width % 8 == 0 && n >= 1 && n <= width);
  TORCH_CHECK(width <= 16384, "lm_post_norm_add: width > 16384");
  if (bias.has_value()) {
    LM_CHECK_CONTIG(*bias);
    TORCH_CHECK(bias->numel() == width &&
                bias->scalar_type() == o.scalar_type());
  }
  const bool own = o.scalar_type() != at::kFloat;
  auto h = own ? torch::empty_like(o) : x;
  if (T == 0) return h;
  const int nv = (width + 2047) / 2048;
#define LM_PN(NV)                                                           \
  hipLaunchKernelGGL((post_norm_add_kernel<scalar_t, NV>), dim3(T),         \
                     dim3(256), 0, cmls::current_stream(),                  \
                     (const scalar_t*)o.data_ptr(),                         \
                     bias.has_value() ? (const scalar_t*)bias->data_ptr()   \
                                      : nullptr,                            \
                     (const scalar_t*)w.data_ptr(), x.data_ptr<float>(),    \
                     own ? (scalar_t*)h.data_ptr() : nullptr, width, (int)n,\
                     (float)eps)
  LM_DISPATCH(o, "lm_post_norm_add", [&] {
    if (nv <= 1) LM_PN(1);
    else if (nv <= 2) LM_PN(2);
    else if (nv <= 4) LM_PN(4);
    else LM_PN(8);
  });
#undef LM_PN
  LM_LAUNCHED();
  return h;
}

torch::Tensor lm_output_norm(torch::Tensor x,
                             c10::optional<torch::Tensor> rows,
                             torch::Tensor w, long n, double eps,
                             double scale) {
  LM_CHECK_CONTIG(x);
  LM_CHECK_CONTIG(w);
  TORCH_CHECK(x.scalar_type() == at::kFloat && x.dim() == 2);
  const int width = x.size(1);
  TORCH_CHECK(w.numel() == width && width % 8 == 0 && n >= 1 && n <= width);
  int R = x.size(0);
  if (rows.has_value()) {
    LM_CHECK_I32(*rows);
    R = rows->numel();
  }
  auto out = torch::empty({R, width}, w.options());
  if (R == 0) return out;
  LM_DISPATCH(w, "lm_output_norm", [&] {
    hipLaunchKernelGGL((output_norm_kernel<scalar_t>), dim3(R), dim3(256), 0,
                       cmls::current_stream(), x.data_ptr<float>(),
                       rows.has_value() ? rows->data_ptr<int>() : nullptr,
                       (const scalar_t*)w.data_ptr(),
                       (scalar_t*)out.data_ptr(), width, (int)n,
                       (int)x.size(0), (float)eps, (float)scale);
  });
  LM_LAUNCHED();
  return out;
}

torch::Tensor lm_gelu_mul(torch::Tensor gu,
                          c10::optional<torch::Tensor> bias) {
  LM_CHECK_CONTIG(gu);
  TORCH_CHECK(gu.dim() == 2 && gu.size(1) % 16 == 0);
  const int T = gu.size(0), ff = gu.size(1) / 2;
  if (bias.has_value()) {
    LM_CHECK_CONTIG(*bias);
    TORCH_CHECK(bias->numel() == 2 * ff &&
                bias->scalar_type() == gu.scalar_type());
  }
  auto out = torch::empty({T, ff}, gu.options());
  if (T == 0) return out;
  LM_DISPATCH(gu, "lm_gelu_mul", [&] {
    hipLaunchKernelGGL((gelu_mul_kernel<scalar_t>),
                       dim3(T, (ff / 8 + 255) / 256), dim3(256), 0,
                       cmls::current_stream(),
                       (const scalar_t*)gu.data_ptr(),
                       bias.has_value() ? (const scalar_t*)bias->data_ptr()
                                        : nullptr,
                       (scalar_t*)out.data_ptr(), ff);
  });
  LM_LAUNCHED();
  return out;
}

torch::Tensor lm_gather_rows(torch::Tensor src, torch::Tensor idx) {
  LM_CHECK_CONTIG(src);
  LM_CHECK_I32(idx);
  const int width = src.size(-1);
  TORCH_CHECK(width % 8 == 0);
  const int n = idx.numel();
  auto out = torch::empty({n, width}, src.options());
  if (n == 0) return out;
  const long total = (long)n * (width / 8);
  LM_DISPATCH(src, "lm_gather_rows", [&] {
    hipLaunchKernelGGL((gather_rows_kernel<scalar_t>),
                       dim3((total + 255) / 256), dim3(256), 0,
                       cmls::current_stream(),
                       (const scalar_t*)src.data_ptr(), idx.data_ptr<int>(),
                       (scalar_t*)out.data_ptr(), n, width,
                       (long)(src.numel() / width));
  });
  LM_LAUNCHED();
  return out;
}
