// Residual-stream kernels: embedding, norm-on-output with residual add, the
// norm in front of the next sublayer, output norm, gated activation.
//
// The residual x is float; each step that changes it also writes what the
// next projection reads (a copy of x, or its norm) in the matrix-product type,
// so x makes one round trip to HBM per sublayer.
//
// Rows are `width` (padded) elements of which `n` count; the pad is zero.
// Norm weights are stored around `off` = 0 or, with off = 1, around zero.
// NV: 8-element vectors of a row that a thread keeps in registers.
#include "lm_common.h"

namespace {

// h = x, or with a weight x / rms(x) * (off + w), for a row in registers
template <typename T, int NV>
__device__ __forceinline__ void write_next(const float (&r)[NV][8],
                                           const T* __restrict__ w, float off,
                                           T* __restrict__ h, int width,
                                           int n, float eps, float* tmp) {
  float inv = 1.f;
  if (w) {
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      if ((i * 256 + (int)threadIdx.x) * 8 < width) {
#pragma unroll
        for (int e = 0; e < 8; ++e) ss += r[i][e] * r[i][e];
      }
    }
    ss = block_reduce(ss, tmp, SumOp{}, 0.f);
    inv = 1.f / sqrtf(ss / (float)n + eps);
  }
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + threadIdx.x) * 8;
    if (c < width) {
      float f[8];
      if (w) {
        load8<T>(w + c, f);
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] = r[i][e] * inv * (off + f[e]);
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] = r[i][e];
      }
      store8(h + c, f);
    }
  }
}

template <typename T, int NV>
__global__ __launch_bounds__(256) void embed_kernel(
    const long* __restrict__ tokens, const T* __restrict__ table,
    float* __restrict__ x, T* __restrict__ h, long ld_h,
    T* __restrict__ copy, long ld_copy, const T* __restrict__ next_w,
    float off, int width, int n, float eps, long vocab) {
  __shared__ float tmp[16];
  const long t = blockIdx.x;
  long id = tokens[t];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  float v[NV][8];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + threadIdx.x) * 8;
    if (c < width) {
      load8<T>(table + id * width + c, v[i]);
      store8(x + t * width + c, v[i]);
      if (copy) store8(copy + t * ld_copy + c, v[i]);
    }
  }
  if (h)
    write_next<T, NV>(v, next_w, off, h + t * ld_h, width, n, eps, tmp);
}

// x += v / rms(v) * (off + w), h from the new x; v = o + bias or, MIX, the
// sum over a token's `top` slots of share * o[pos]
template <typename T, int NV, bool MIX>
__global__ __launch_bounds__(256) void post_norm_add_kernel(
    const T* __restrict__ o, const T* __restrict__ bias,
    const int* __restrict__ pos, const float* __restrict__ share, int top,
    int n_rows, const T* __restrict__ w, float off, float* __restrict__ x,
    const T* __restrict__ next_w, T* __restrict__ h, long ld_h, int width,
    int n, float eps) {
  __shared__ float tmp[16];
  __shared__ float tmp2[16];
  const long t = blockIdx.x, row = t * width;
  float v[NV][8];
  float ss = 0.f;
  if (MIX) {
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
      for (int e = 0; e < 8; ++e) v[i][e] = 0.f;
    for (int k = 0; k < top; ++k) {
      const long p = min(max(pos[t * top + k], 0), n_rows - 1);
      const float s = share[t * top + k];
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int c = (i * 256 + threadIdx.x) * 8;
        if (c < width) {
          float f[8];
          load8<T>(o + p * width + c, f);
#pragma unroll
          for (int e = 0; e < 8; ++e) v[i][e] += s * f[e];
        }
      }
    }
  }
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + threadIdx.x) * 8;
    if (c < width) {
      if (!MIX) load8<T>(o + row + c, v[i]);
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
      for (int e = 0; e < 8; ++e) v[i][e] = r[e] + v[i][e] * inv * (off + g[e]);
      store8(x + row + c, v[i]);
    }
  }
  if (h)
    write_next<T, NV>(v, next_w, off, h + t * ld_h, width, n, eps, tmp2);
}

// h = r / rms(r) * w for one or two weights of a row in registers
template <typename T, int NV>
__device__ __forceinline__ void write_norms(
    const float (&r)[NV][8], const T* __restrict__ wa, T* __restrict__ ha,
    const T* __restrict__ wb, T* __restrict__ hb, int width, int n, float eps,
    float* tmp) {
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    if ((i * 256 + (int)threadIdx.x) * 8 < width) {
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += r[i][e] * r[i][e];
    }
  }
  ss = block_reduce(ss, tmp, SumOp{}, 0.f);
  const float inv = 1.f / sqrtf(ss / (float)n + eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + threadIdx.x) * 8;
    if (c >= width) continue;
    float f[8];
    load8<T>(wa + c, f);
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] *= r[i][e] * inv;
    store8(ha + c, f);
    if (wb) {
      load8<T>(wb + c, f);
#pragma unroll
      for (int e = 0; e < 8; ++e) f[e] *= r[i][e] * inv;
      store8(hb + c, f);
    }
  }
}

template <typename T, int NV>
__global__ __launch_bounds__(256) void embed_norms_kernel(
    const long* __restrict__ tokens, const T* __restrict__ table,
    float* __restrict__ x, const T* __restrict__ wa, T* __restrict__ ha,
    const T* __restrict__ wb, T* __restrict__ hb, int width, int n, float eps,
    long vocab) {
  __shared__ float tmp[16];
  const long row = (long)blockIdx.x * width;
  long id = tokens[blockIdx.x];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  float v[NV][8];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + threadIdx.x) * 8;
    if (c < width) {
      load8<T>(table + id * width + c, v[i]);
      store8(x + row + c, v[i]);
    }
  }
  write_norms<T, NV>(v, wa, ha + row, wb, wb ? hb + row : nullptr, width, n,
                     eps, tmp);
}

// What parallel sublayers made goes into the stream: x += plain + scale *
// (o1 / rms(o1) * w1 + o2 / rms(o2) * w2), each part optional; up to two norms
// of the new x. Two sums are reduced at once.
template <typename T, int NV, bool BR>
__global__ __launch_bounds__(256) void add_branches_kernel(
    float* __restrict__ x, const T* __restrict__ plain,
    const T* __restrict__ o1, const T* __restrict__ w1,
    const T* __restrict__ o2, const T* __restrict__ w2, float scale,
    const T* __restrict__ wa, T* __restrict__ ha, const T* __restrict__ wb,
    T* __restrict__ hb, int width, int n, float eps) {
  __shared__ float tmp[16];
  __shared__ float sums[2][4];
  const long row = (long)blockIdx.x * width;
  const int tid = threadIdx.x;
  float v[NV][8], f1[BR ? NV : 1][8], f2[BR ? NV : 1][8];
  float s1 = 0.f, s2 = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + tid) * 8;
    if (c >= width) continue;
    load8<float>(x + row + c, v[i]);
    if (plain) {
      float p[8];
      load8<T>(plain + row + c, p);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[i][e] += p[e];
    }
    if (BR) {
      load8<T>(o1 + row + c, f1[BR ? i : 0]);
#pragma unroll
      for (int e = 0; e < 8; ++e) s1 += f1[BR ? i : 0][e] * f1[BR ? i : 0][e];
      if (o2) {
        load8<T>(o2 + row + c, f2[BR ? i : 0]);
#pragma unroll
        for (int e = 0; e < 8; ++e)
          s2 += f2[BR ? i : 0][e] * f2[BR ? i : 0][e];
      }
    }
  }
  if (BR) {
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      s1 += __shfl_xor(s1, d, 64);
      s2 += __shfl_xor(s2, d, 64);
    }
    if ((tid & 63) == 0) {
      sums[0][tid >> 6] = s1;
      sums[1][tid >> 6] = s2;
    }
    __syncthreads();
    s1 = (sums[0][0] + sums[0][1]) + (sums[0][2] + sums[0][3]);
    s2 = (sums[1][0] + sums[1][1]) + (sums[1][2] + sums[1][3]);
    s1 = scale / sqrtf(s1 / (float)n + eps);
    s2 = scale / sqrtf(s2 / (float)n + eps);
  }
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + tid) * 8;
    if (c >= width) continue;
    if (BR) {
      float g[8];
      load8<T>(w1 + c, g);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[i][e] += f1[BR ? i : 0][e] * s1 * g[e];
      if (o2) {
        load8<T>(w2 + c, g);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[i][e] += f2[BR ? i : 0][e] * s2 * g[e];
      }
    }
    store8(x + row + c, v[i]);
  }
  if (wa)
    write_norms<T, NV>(v, wa, ha + row, wb, wb ? hb + row : nullptr, width, n,
                       eps, tmp);
}

// z > 0: a z^2 + z / 2, else b (e^z - 1 - z) + z / 2
__device__ __forceinline__ float xielu_f(float z, float a, float b) {
  // e^z - 1 - z: the power series where the difference would cancel
  const float p = z * z *
      (1.f / 2 + z * (1.f / 6 + z * (1.f / 24 + z * (1.f / 120 +
       z * (1.f / 720 + z * (1.f / 5040))))));
  const float d = z > -0.5f ? p : exp_f(z) - 1.f - z;
  return (z > 0.f ? a * z * z : b * d) + 0.5f * z;
}

template <typename T>
__global__ __launch_bounds__(256) void xielu_kernel(
    const T* __restrict__ z, const float* __restrict__ coef,
    T* __restrict__ out, long ld_out, int ff, long total) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const int per = ff / 8;
  const long t = i / per;
  const int c = (int)(i % per) * 8;
  const float a = coef[0], b = coef[1];
  float f[8];
  load8<T>(z + t * ff + c, f);
#pragma unroll
  for (int e = 0; e < 8; ++e) f[e] = xielu_f(f[e], a, b);
  store8(out + t * ld_out + c, f);
}

// x += add (one vector for all rows); h from the new x
template <typename T, int NV>
__global__ __launch_bounds__(256) void add_norm_kernel(
    float* __restrict__ x, const T* __restrict__ add,
    const T* __restrict__ next_w, float off, T* __restrict__ h, int width,
    int n, float eps) {
  __shared__ float tmp[16];
  const long row = (long)blockIdx.x * width;
  float v[NV][8];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * 256 + threadIdx.x) * 8;
    if (c < width) {
      float a[8];
      load8<T>(add + c, a);
      load8<float>(x + row + c, v[i]);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[i][e] += a[e];
      store8(x + row + c, v[i]);
    }
  }
  write_next<T, NV>(v, next_w, off, h + row, width, n, eps, tmp);
}

// out[i] = norm(x[rows[i]]) * (off + w) * scale
template <typename T>
__global__ __launch_bounds__(256) void output_norm_kernel(
    const float* __restrict__ x, const int* __restrict__ rows,
    const T* __restrict__ w, T* __restrict__ out, int width, int n,
    int n_tok, float eps, float scale, float off) {
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
    for (int e = 0; e < 8; ++e) f[e] = f[e] * inv * (off + g[e]) * scale;
    store8(out + (long)blockIdx.x * width + c, f);
  }
}

// gu = [gate | up] rows of 2*ff; out = act(gate + bg) * (up + bu)
template <typename T, int ACT>
__global__ __launch_bounds__(256) void gated_mul_kernel(
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
  for (int e = 0; e < 8; ++e) g[e] = act_f<ACT>(g[e]) * u[e];
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

// rows of 8-element vectors per thread -> template argument NV
#define LM_NV(WIDTH, CALL)                         \
  do {                                             \
    const int nv_ = ((WIDTH) + 2047) / 2048;       \
    if (nv_ <= 1) { CALL(1); }                     \
    else if (nv_ <= 2) { CALL(2); }                \
    else if (nv_ <= 4) { CALL(4); }                \
    else { CALL(8); }                              \
  } while (0)

// [T, width] view whose rows are 16-byte aligned; -> row stride
static long row_view(const torch::Tensor& v, long rows, long width,
                     at::ScalarType type) {
  TORCH_CHECK(v.is_cuda() && v.dim() == 2 && v.size(0) == rows &&
                  v.size(1) == width && v.stride(1) == 1 &&
                  v.stride(0) % 8 == 0 && v.storage_offset() % 8 == 0 &&
                  v.scalar_type() == type,
              "lm: output rows do not fit");
  return v.stride(0);
}

static void check_weight(const c10::optional<torch::Tensor>& w, long width,
                         at::ScalarType type) {
  if (!w.has_value()) return;
  LM_CHECK_CONTIG(*w);
  TORCH_CHECK(w->numel() == width && w->scalar_type() == type);
}

// -> {x, h}. h: the next projection's input, into `out` if given; `copy`
// receives the rows as they are.
std::vector<torch::Tensor> lm_embed(torch::Tensor tokens, torch::Tensor table,
                                    c10::optional<torch::Tensor> next_w,
                                    double off, long n, double eps,
                                    c10::optional<torch::Tensor> out,
                                    c10::optional<torch::Tensor> copy) {
  LM_CHECK_CONTIG(tokens);
  LM_CHECK_CONTIG(table);
  TORCH_CHECK(tokens.scalar_type() == at::kLong && tokens.dim() == 1);
  const int T = tokens.size(0), width = table.size(1);
  TORCH_CHECK(width % 8 == 0 && width <= 16384, "lm_embed: width");
  TORCH_CHECK(n >= 1 && n <= width);
  const auto type = table.scalar_type();
  check_weight(next_w, width, type);
  auto x = torch::empty({T, width}, table.options().dtype(at::kFloat));
  // in 32-bit runs the stream itself can be the projection input
  const bool alias = type == at::kFloat && !next_w && !out;
  auto h = out ? *out : alias ? x : torch::empty({T, width}, table.options());
  const long ld_h = row_view(h, T, width, type);
  const long ld_c = copy ? row_view(*copy, T, width, type) : 0;
  if (T == 0) return {x, h};
#define LM_EMBED(NV)                                                         \
  hipLaunchKernelGGL((embed_kernel<scalar_t, NV>), dim3(T), dim3(256), 0,    \
                     cmls::current_stream(), tokens.data_ptr<long>(),        \
                     (const scalar_t*)table.data_ptr(), x.data_ptr<float>(), \
                     alias ? nullptr : (scalar_t*)h.data_ptr(), ld_h,        \
                     copy ? (scalar_t*)copy->data_ptr() : nullptr, ld_c,     \
                     next_w ? (const scalar_t*)next_w->data_ptr() : nullptr, \
                     (float)off, width, (int)n, (float)eps,                  \
                     (long)table.size(0))
  LM_DISPATCH(table, "lm_embed", [&] { LM_NV(width, LM_EMBED); });
#undef LM_EMBED
  LM_LAUNCHED();
  return {x, h};
}

// o: [T, width], or with pos, share [T, top] the rows they pick and weigh
torch::Tensor lm_post_norm_add(torch::Tensor o,
                               c10::optional<torch::Tensor> bias,
                               torch::Tensor w, torch::Tensor x, long n,
                               double eps, double off,
                               c10::optional<torch::Tensor> next_w,
                               c10::optional<torch::Tensor> out,
                               c10::optional<torch::Tensor> pos,
                               c10::optional<torch::Tensor> share) {
  LM_CHECK_CONTIG(o);
  LM_CHECK_CONTIG(w);
  LM_CHECK_CONTIG(x);
  TORCH_CHECK(o.dim() == 2 && x.dim() == 2);
  const int T = x.size(0), width = x.size(1);
  const auto type = o.scalar_type();
  TORCH_CHECK(x.scalar_type() == at::kFloat && o.size(1) == width);
  TORCH_CHECK(w.numel() == width && w.scalar_type() == type);
  TORCH_CHECK(width % 8 == 0 && n >= 1 && n <= width);
  TORCH_CHECK(width <= 16384, "lm_post_norm_add: width > 16384");
  check_weight(bias, width, type);
  check_weight(next_w, width, type);
  int top = 0;
  if (pos) {
    TORCH_CHECK(share.has_value());
    LM_CHECK_I32(*pos);
    LM_CHECK_CONTIG(*share);
    TORCH_CHECK(pos->dim() == 2 && pos->size(0) == T &&
                share->sizes() == pos->sizes() &&
                share->scalar_type() == at::kFloat);
    TORCH_CHECK(T == 0 || o.size(0) > 0);
    top = pos->size(1);
  } else {
    TORCH_CHECK(o.size(0) == T);
  }
  const bool alias = type == at::kFloat && !next_w && !out;
  auto h = out ? *out : alias ? x : torch::empty({T, width}, o.options());
  const long ld_h = row_view(h, T, width, type);
  if (T == 0) return h;
#define LM_PN_(NV, MIX)                                                     \
  hipLaunchKernelGGL((post_norm_add_kernel<scalar_t, NV, MIX>), dim3(T),    \
                     dim3(256), 0, cmls::current_stream(),                  \
                     (const scalar_t*)o.data_ptr(),                         \
                     bias ? (const scalar_t*)bias->data_ptr() : nullptr,    \
                     pos ? pos->data_ptr<int>() : nullptr,                  \
                     share ? share->data_ptr<float>() : nullptr, top,       \
                     (int)o.size(0), (const scalar_t*)w.data_ptr(),         \
                     (float)off, x.data_ptr<float>(),                       \
                     next_w ? (const scalar_t*)next_w->data_ptr() : nullptr,\
                     alias ? nullptr : (scalar_t*)h.data_ptr(), ld_h,       \
                     width, (int)n, (float)eps)
#define LM_PN(NV) do { if (pos) LM_PN_(NV, true); else LM_PN_(NV, false); } while (0)
  LM_DISPATCH(o, "lm_post_norm_add", [&] { LM_NV(width, LM_PN); });
#undef LM_PN
#undef LM_PN_
  LM_LAUNCHED();
  return h;
}

torch::Tensor lm_add_norm(torch::Tensor x, torch::Tensor add,
                          c10::optional<torch::Tensor> next_w, double off,
                          long n, double eps) {
  LM_CHECK_CONTIG(x);
  LM_CHECK_CONTIG(add);
  TORCH_CHECK(x.scalar_type() == at::kFloat && x.dim() == 2);
  const int T = x.size(0), width = x.size(1);
  TORCH_CHECK(add.numel() == width && width % 8 == 0 && width <= 16384);
  TORCH_CHECK(n >= 1 && n <= width);
  check_weight(next_w, width, add.scalar_type());
  auto h = torch::empty({T, width}, add.options());
  if (T == 0) return h;
#define LM_AN(NV)                                                           \
  hipLaunchKernelGGL((add_norm_kernel<scalar_t, NV>), dim3(T), dim3(256),   \
                     0, cmls::current_stream(), x.data_ptr<float>(),        \
                     (const scalar_t*)add.data_ptr(),                       \
                     next_w ? (const scalar_t*)next_w->data_ptr() : nullptr,\
                     (float)off, (scalar_t*)h.data_ptr(), width, (int)n,    \
                     (float)eps)
  LM_DISPATCH(add, "lm_add_norm", [&] { LM_NV(width, LM_AN); });
#undef LM_AN
  LM_LAUNCHED();
  return h;
}

// -> {x, norm of x for each of one or two weights}
std::vector<torch::Tensor> lm_embed_norms(torch::Tensor tokens,
                                          torch::Tensor table,
                                          torch::Tensor wa,
                                          c10::optional<torch::Tensor> wb,
                                          long n, double eps) {
  LM_CHECK_CONTIG(tokens);
  LM_CHECK_CONTIG(table);
  TORCH_CHECK(tokens.scalar_type() == at::kLong && tokens.dim() == 1);
  const int T = tokens.size(0), width = table.size(1);
  TORCH_CHECK(table.dim() == 2 && width % 8 == 0 && width <= 16384 &&
              table.size(0) > 0);
  TORCH_CHECK(n >= 1 && n <= width);
  const auto type = table.scalar_type();
  check_weight(wa, width, type);
  check_weight(wb, width, type);
  std::vector<torch::Tensor> out{
      torch::empty({T, width}, table.options().dtype(at::kFloat)),
      torch::empty({T, width}, table.options())};
  if (wb) out.push_back(torch::empty({T, width}, table.options()));
  if (T == 0) return out;
#define LM_EN(NV)                                                            \
  hipLaunchKernelGGL((embed_norms_kernel<scalar_t, NV>), dim3(T), dim3(256), \
                     0, cmls::current_stream(), tokens.data_ptr<long>(),     \
                     (const scalar_t*)table.data_ptr(),                      \
                     out[0].data_ptr<float>(),                               \
                     (const scalar_t*)wa.data_ptr(),                         \
                     (scalar_t*)out[1].data_ptr(),                           \
                     wb ? (const scalar_t*)wb->data_ptr() : nullptr,         \
                     wb ? (scalar_t*)out[2].data_ptr() : nullptr, width,     \
                     (int)n, (float)eps, (long)table.size(0))
  LM_DISPATCH(table, "lm_embed_norms", [&] { LM_NV(width, LM_EN); });
#undef LM_EN
  LM_LAUNCHED();
  return out;
}

// x float [T, width] in place; plain, o1, o2 [T, width]; -> norms of the new x
std::vector<torch::Tensor> lm_add_branches(
    torch::Tensor x, c10::optional<torch::Tensor> plain,
    c10::optional<torch::Tensor> o1, c10::optional<torch::Tensor> w1,
    c10::optional<torch::Tensor> o2, c10::optional<torch::Tensor> w2,
    double scale, c10::optional<torch::Tensor> wa,
    c10::optional<torch::Tensor> wb, long n, double eps) {
  LM_CHECK_CONTIG(x);
  TORCH_CHECK(x.scalar_type() == at::kFloat && x.dim() == 2);
  const int T = x.size(0), width = x.size(1);
  TORCH_CHECK(width % 8 == 0 && width <= 16384 && n >= 1 && n <= width);
  TORCH_CHECK(plain || o1, "lm_add_branches: nothing to add");
  const auto type = (plain ? *plain : *o1).scalar_type();
  for (const auto* o : {&plain, &o1, &o2})
    if (o->has_value()) {
      LM_CHECK_CONTIG(**o);
      TORCH_CHECK((*o)->sizes() == x.sizes() && (*o)->scalar_type() == type);
    }
  TORCH_CHECK(o1.has_value() == w1.has_value() &&
              o2.has_value() == w2.has_value() && (o1 || !o2) && (wa || !wb));
  for (const auto* w : {&w1, &w2, &wa, &wb}) check_weight(*w, width, type);
  std::vector<torch::Tensor> out;
  const auto opt = x.options().dtype(type);
  if (wa) out.push_back(torch::empty({T, width}, opt));
  if (wb) out.push_back(torch::empty({T, width}, opt));
  if (T == 0) return out;
#define LM_PTR(V) (V ? (const scalar_t*)V->data_ptr() : nullptr)
#define LM_AB_(NV, BR)                                                       \
  hipLaunchKernelGGL((add_branches_kernel<scalar_t, NV, BR>), dim3(T),       \
                     dim3(256), 0, cmls::current_stream(),                   \
                     x.data_ptr<float>(), LM_PTR(plain), LM_PTR(o1),         \
                     LM_PTR(w1), LM_PTR(o2), LM_PTR(w2), (float)scale,       \
                     LM_PTR(wa), wa ? (scalar_t*)out[0].data_ptr() : nullptr,\
                     LM_PTR(wb), wb ? (scalar_t*)out[1].data_ptr() : nullptr,\
                     width, (int)n, (float)eps)
#define LM_AB(NV) do { if (o1) LM_AB_(NV, true); else LM_AB_(NV, false); } while (0)
  auto& of = plain ? *plain : *o1;
  LM_DISPATCH(of, "lm_add_branches", [&] { LM_NV(width, LM_AB); });
#undef LM_AB
#undef LM_AB_
#undef LM_PTR
  LM_LAUNCHED();
  return out;
}

// coef float (a, b); out [T, ff], row stride free
void lm_xielu(torch::Tensor z, torch::Tensor coef, torch::Tensor out) {
  LM_CHECK_CONTIG(z);
  LM_CHECK_CONTIG(coef);
  TORCH_CHECK(z.dim() == 2 && z.size(1) % 8 == 0);
  TORCH_CHECK(coef.numel() == 2 && coef.scalar_type() == at::kFloat);
  const int ff = z.size(1);
  const long ld = row_view(out, z.size(0), ff, z.scalar_type());
  const long total = z.numel() / 8;
  if (total == 0) return;
  LM_DISPATCH(z, "lm_xielu", [&] {
    hipLaunchKernelGGL((xielu_kernel<scalar_t>), dim3((total + 255) / 256),
                       dim3(256), 0, cmls::current_stream(),
                       (const scalar_t*)z.data_ptr(), coef.data_ptr<float>(),
                       (scalar_t*)out.data_ptr(), ld, ff, total);
  });
  LM_LAUNCHED();
}

torch::Tensor lm_output_norm(torch::Tensor x,
                             c10::optional<torch::Tensor> rows,
                             torch::Tensor w, long n, double eps,
                             double scale, double off) {
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
                       (int)x.size(0), (float)eps, (float)scale, (float)off);
  });
  LM_LAUNCHED();
  return out;
}

// act: 0 tanh-form GELU, 1 SiLU
torch::Tensor lm_gated_mul(torch::Tensor gu, c10::optional<torch::Tensor> bias,
                           long act) {
  LM_CHECK_CONTIG(gu);
  TORCH_CHECK(gu.dim() == 2 && gu.size(1) % 16 == 0);
  TORCH_CHECK(act == LM_GELU_TANH || act == LM_SILU);
  const int T = gu.size(0), ff = gu.size(1) / 2;
  check_weight(bias, 2 * ff, gu.scalar_type());
  auto out = torch::empty({T, ff}, gu.options());
  if (T == 0) return out;
#define LM_GM(ACT)                                                          \
  hipLaunchKernelGGL((gated_mul_kernel<scalar_t, ACT>),                     \
                     dim3(T, (ff / 8 + 255) / 256), dim3(256), 0,           \
                     cmls::current_stream(), (const scalar_t*)gu.data_ptr(),\
                     bias ? (const scalar_t*)bias->data_ptr() : nullptr,    \
                     (scalar_t*)out.data_ptr(), ff)
  LM_DISPATCH(gu, "lm_gated_mul", [&] {
    if (act == LM_SILU) LM_GM(LM_SILU);
    else LM_GM(LM_GELU_TANH);
  });
#undef LM_GM
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
