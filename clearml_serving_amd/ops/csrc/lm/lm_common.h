// Shared pieces of the token-batch kernels (csrc/lm).
//
// Every operand the kernels see is padded: feature dimensions are multiples
// of 32 with zeros behind the true size, so there are no tails in any inner
// loop. Kernels are templated on the storage type: bf16 for serving, float
// for exact 32-bit runs; accumulation is always float.
#pragma once

#include "../common.h"

typedef __hip_bfloat16 bf16;
typedef __attribute__((ext_vector_type(8))) short lm_s16x8;
typedef __attribute__((ext_vector_type(4))) short lm_s16x4;
typedef __attribute__((ext_vector_type(4))) float lm_f32x4;

// Eight consecutive k-elements of one operand row. For a 16x16x32 product,
// lane l holds row (l & 15), k = (l >> 4) * 8 + [0, 8).
template <typename T> struct Frag;
template <> struct Frag<bf16> { lm_s16x8 v; };
template <> struct Frag<float> { float v[8]; };

__device__ __forceinline__ Frag<bf16> load_frag(const bf16* p) {
  Frag<bf16> f;
  f.v = *reinterpret_cast<const lm_s16x8*>(p);
  return f;
}
__device__ __forceinline__ Frag<float> load_frag(const float* p) {
  Frag<float> f;
  const lm_f32x4 lo = *reinterpret_cast<const lm_f32x4*>(p);
  const lm_f32x4 hi = *reinterpret_cast<const lm_f32x4*>(p + 4);
#pragma unroll
  for (int e = 0; e < 4; ++e) { f.v[e] = lo[e]; f.v[4 + e] = hi[e]; }
  return f;
}
// Operands whose k runs down the rows of an LDS tile. k order of the eight
// slots of lane group g: rows 4g..4g+3, then 16+4g..16+4g+3 -- the order in
// which a 16x16 result holds its rows, so a result register file is directly
// the other operand. Column = lane & 15.
typedef __attribute__((address_space(3))) lm_s16x4 lm_lds_s16x4;
__device__ __forceinline__ Frag<bf16> load_frag_rows(const bf16* tile,
                                                     int pitch) {
  // ds_read_b64_tr_b16: a 16-lane group reads 4 rows x 16 columns, lane i
  // supplying row i/4, columns 4*(i%4)..+3, and receives column i
  const int lane = threadIdx.x & 63, i = lane & 15;
  const bf16* p = tile + (4 * (lane >> 4) + (i >> 2)) * pitch + (i & 3) * 4;
  const lm_s16x4 lo =
      __builtin_amdgcn_ds_read_tr16_b64_v4i16((lm_lds_s16x4*)p);
  const lm_s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (lm_lds_s16x4*)(p + 16 * pitch));
  Frag<bf16> f;
  f.v = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
  return f;
}
__device__ __forceinline__ Frag<float> load_frag_rows(const float* tile,
                                                      int pitch) {
  const int lane = threadIdx.x & 63;
  const float* p = tile + 4 * (lane >> 4) * pitch + (lane & 15);
  Frag<float> f;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    f.v[e] = p[e * pitch];
    f.v[4 + e] = p[(16 + e) * pitch];
  }
  return f;
}
// the operand made of two such results (rows 0..15 and 16..31)
template <typename T>
__device__ __forceinline__ Frag<T> frag_of(const lm_f32x4& lo,
                                           const lm_f32x4& hi);
template <>
__device__ __forceinline__ Frag<bf16> frag_of<bf16>(const lm_f32x4& lo,
                                                    const lm_f32x4& hi) {
  union { lm_s16x8 v; bf16 b[8]; } u;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    u.b[e] = __float2bfloat16(lo[e]);
    u.b[4 + e] = __float2bfloat16(hi[e]);
  }
  Frag<bf16> f;
  f.v = u.v;
  return f;
}
template <>
__device__ __forceinline__ Frag<float> frag_of<float>(const lm_f32x4& lo,
                                                      const lm_f32x4& hi) {
  Frag<float> f;
#pragma unroll
  for (int e = 0; e < 4; ++e) { f.v[e] = lo[e]; f.v[4 + e] = hi[e]; }
  return f;
}
// LDS traffic between the lanes of one wave: order it without a barrier
__device__ __forceinline__ void wave_lds_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}
// The wave's number, as a scalar. An MFMA ignores the lane mask, so a branch
// around one has to be a scalar branch.
__device__ __forceinline__ int uniform_wave() {
  return __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
}
template <typename T> __device__ __forceinline__ Frag<T> zero_frag();
template <> __device__ __forceinline__ Frag<bf16> zero_frag<bf16>() {
  Frag<bf16> f;
  f.v = lm_s16x8{0, 0, 0, 0, 0, 0, 0, 0};
  return f;
}
template <> __device__ __forceinline__ Frag<float> zero_frag<float>() {
  Frag<float> f;
#pragma unroll
  for (int e = 0; e < 8; ++e) f.v[e] = 0.f;
  return f;
}

// c[4*(l>>4)+r][l&15] += sum over 32 k of a-row times b-row
__device__ __forceinline__ lm_f32x4 mma32(const Frag<bf16>& a,
                                          const Frag<bf16>& b, lm_f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
}
// The fp32 unit takes 4 k per instruction, one per lane group: step e covers
// k = {e, 8+e, 16+e, 24+e}, so eight steps cover the same 32.
__device__ __forceinline__ lm_f32x4 mma32(const Frag<float>& a,
                                          const Frag<float>& b, lm_f32x4 c) {
#pragma unroll
  for (int e = 0; e < 8; ++e)
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.v[e], b.v[e], c, 0, 0, 0);
  return c;
}

// 8-element vector access
template <typename T>
__device__ __forceinline__ void load8(const T* p, float* f);
template <>
__device__ __forceinline__ void load8<bf16>(const bf16* p, float* f) {
  bf16x8 u;
  u.u = *reinterpret_cast<const uint32x4*>(p);
#pragma unroll
  for (int e = 0; e < 8; ++e) f[e] = to_f32(u.h[e]);
}
template <>
__device__ __forceinline__ void load8<float>(const float* p, float* f) {
  const lm_f32x4 lo = *reinterpret_cast<const lm_f32x4*>(p);
  const lm_f32x4 hi = *reinterpret_cast<const lm_f32x4*>(p + 4);
#pragma unroll
  for (int e = 0; e < 4; ++e) { f[e] = lo[e]; f[4 + e] = hi[e]; }
}
__device__ __forceinline__ void store8(bf16* p, const float* f) {
  bf16x8 u;
#pragma unroll
  for (int e = 0; e < 8; ++e) u.h[e] = __float2bfloat16(f[e]);
  *reinterpret_cast<uint32x4*>(p) = u.u;
}
__device__ __forceinline__ void store8(float* p, const float* f) {
  *reinterpret_cast<lm_f32x4*>(p) = lm_f32x4{f[0], f[1], f[2], f[3]};
  *reinterpret_cast<lm_f32x4*>(p + 4) = lm_f32x4{f[4], f[5], f[6], f[7]};
}
__device__ __forceinline__ void store4(bf16* p, const float* f) {
  union { uint2 u; bf16 h[4]; } o;
#pragma unroll
  for (int e = 0; e < 4; ++e) o.h[e] = __float2bfloat16(f[e]);
  *reinterpret_cast<uint2*>(p) = o.u;
}
__device__ __forceinline__ void store4(float* p, const float* f) {
  *reinterpret_cast<lm_f32x4*>(p) = lm_f32x4{f[0], f[1], f[2], f[3]};
}
// copy 8 elements without touching their bits
__device__ __forceinline__ void copy8(bf16* d, const bf16* s) {
  *reinterpret_cast<uint32x4*>(d) = *reinterpret_cast<const uint32x4*>(s);
}
__device__ __forceinline__ void copy8(float* d, const float* s) {
  reinterpret_cast<uint32x4*>(d)[0] = reinterpret_cast<const uint32x4*>(s)[0];
  reinterpret_cast<uint32x4*>(d)[1] = reinterpret_cast<const uint32x4*>(s)[1];
}
__device__ __forceinline__ void zero8(bf16* d) {
  *reinterpret_cast<uint32x4*>(d) = uint32x4{0u, 0u, 0u, 0u};
}
__device__ __forceinline__ void zero8(float* d) {
  reinterpret_cast<uint32x4*>(d)[0] = uint32x4{0u, 0u, 0u, 0u};
  reinterpret_cast<uint32x4*>(d)[1] = uint32x4{0u, 0u, 0u, 0u};
}

// v_exp_f32 and v_rcp_f32: full float, within about 1 ulp
__device__ __forceinline__ float exp_f(float z) {
  return __builtin_amdgcn_exp2f(z * 1.4426950408889634f);
}
__device__ __forceinline__ float sigmoid_f(float z) {
  return __builtin_amdgcn_rcpf(1.f + exp_f(-z));
}
// tanh form: 0.5 z (1 + tanh k) = z * sigmoid(2 k)
__device__ __forceinline__ float gelu_tanh_f(float z) {
  const float k = 0.7978845608028654f * (z + 0.044715f * z * z * z);
  return z * sigmoid_f(2.f * k);
}
// activations that kernels take as a template argument
enum {
  LM_GELU_TANH = 0, LM_SILU = 1, LM_RELU2 = 2, LM_NO_ACT = 3,
  LM_SWIGLU = 4  // gated products: silu(gate) * up of column pairs
};
template <int ACT> __device__ __forceinline__ float act_f(float z) {
  if (ACT == LM_GELU_TANH) return gelu_tanh_f(z);
  if (ACT == LM_SILU) return z * sigmoid_f(z);
  if (ACT == LM_RELU2) return z > 0.f ? z * z : 0.f;
  return z;
}
// 1 - exp(v) for v <= 0: the power series where the difference would cancel
__device__ __forceinline__ float one_minus_exp_f(float v) {
  const float p =
      1.f + v * (1.f / 2 + v * (1.f / 6 + v * (1.f / 24 +
            v * (1.f / 120 + v * (1.f / 720)))));
  return v > -0.25f ? -v * p : 1.f - exp_f(v);
}
__device__ __forceinline__ float softplus_f(float z) {
  return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));
}

#define LM_DISPATCH(TENSOR, NAME, ...)                                     \
  [&] {                                                                    \
    if ((TENSOR).scalar_type() == at::kBFloat16) {                         \
      using scalar_t = __hip_bfloat16;                                     \
      return __VA_ARGS__();                                                \
    } else if ((TENSOR).scalar_type() == at::kFloat) {                     \
      using scalar_t = float;                                              \
      return __VA_ARGS__();                                                \
    }                                                                      \
    TORCH_CHECK(false, NAME, ": bf16 or fp32 only");                       \
  }()

#define LM_CHECK_CUDA(x) TORCH_CHECK((x).is_cuda(), #x " must be on the GPU")
#define LM_CHECK_CONTIG(x) \
  TORCH_CHECK((x).is_cuda() && (x).is_contiguous(), #x " must be contiguous")
#define LM_CHECK_I32(x)                                             \
  TORCH_CHECK((x).is_cuda() && (x).scalar_type() == at::kInt &&     \
                  (x).is_contiguous(),                              \
              #x " must be contiguous int32 on the GPU")
#define LM_LAUNCHED() HIP_CHECK(hipGetLastError())
