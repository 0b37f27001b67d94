// Latent attention: one cached latent c (plus one rotated key part) per
// token, shared by all heads.
//
// Cache row = [c, padded to CP | rotated key part, padded to RP], in pages of
// block_size rows. Two ways to attend to it:
//
// - absorbed (few queries per sequence): q' = [W_uk^T q | q_rot] per head, so
//   every head scores against the cache row itself and sums rows of c; W_uv
//   follows. Reads each cached row once for all heads of a workgroup.
// - expanded (prompts): keys and values are rebuilt per head from the rows a
//   portion can see, then ordinary flash attention runs on them; several
//   times fewer multiply-adds when kv_rank exceeds the head size.
//
// Both take a sliding window, a per-head sink (a term exp(sink) in the softmax
// denominator that has no key) and a gate on the heads' outputs, each of them
// optional. Queries may come from a normed latent of their own.
#include "lm_attn.h"

namespace {

// ------------------------------------------------------------------- //
// prepare: rotate q; normalise the query latent and the cached latent, rotate
// the shared key part, write the cache row. Each part is optional.
// ------------------------------------------------------------------- //
template <typename T>
struct PrepArgs {
  T* q;            // [t, heads * (DP + RP)], rows of ldq; null: no q here
  long ldq;
  int heads, DP;
  T* q_abs;        // rotated part of the first n_abs tokens goes here
  int n_abs;
  const T* lat;    // [t, CP + RP], rows of ld_lat; null: no latent here
  long ld_lat;
  const T* kv_norm;
  int kv_rank;
  T* cache;
  long n_slots;
  const T* cq;     // [t, QP], rows of ld_lat; null: no query latent
  const T* q_norm;
  T* cq_out;
  int QP, q_rank;
};

// dst = v / rms(v) * w by one wave; `count` of the `n` elements are real
template <typename T>
__device__ __forceinline__ void wave_norm(T* dst, const T* v, const T* w,
                                          int n, int count, float eps) {
  const int lane = threadIdx.x & 63;
  float ss = 0.f;
  for (int c = lane * 8; c < n; c += 64 * 8) {
    float f[8];
    load8<T>(v + c, f);
#pragma unroll
    for (int e = 0; e < 8; ++e) ss += f[e] * f[e];
  }
  const float inv = 1.f / sqrtf(wave_reduce_sum(ss) / (float)count + eps);
  for (int c = lane * 8; c < n; c += 64 * 8) {
    float f[8], g[8];
    load8<T>(v + c, f);
    load8<T>(w + c, g);
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] = f[e] * inv * g[e];
    store8(dst + c, f);
  }
}

// one wave per token
constexpr int PREP_W = 4;

template <typename T>
__global__ __launch_bounds__(PREP_W * 64) void latent_prep_kernel(
    PrepArgs<T> a, const int* __restrict__ positions,
    const int* __restrict__ slots, Rot rot, int RP, int CP, float eps,
    int n_tok) {
  __shared__ float trig[PREP_W][2][256];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int t = blockIdx.x * PREP_W + wave;
  if (t >= n_tok) return;  // no barrier below
  float* cs = trig[wave][0];
  float* sn = trig[wave][1];
  const int pairs = rot.pairs;
  const float pos = (float)positions[t];
  for (int i = lane; i < pairs; i += 64) {
    float s, c;
    sincosf(pos * rot.inv_freq[i], &s, &c);
    cs[i] = rot.gain * c;
    sn[i] = rot.gain * s;
  }
  wave_lds_fence();
  const int hp = RP / 2;
  if (a.q) {
    T* row = a.q + (long)t * a.ldq;
    const bool absorbed = t < a.n_abs;
    const int q_pairs = absorbed ? hp : pairs;  // the rest passes unchanged
    for (int i = lane; i < a.heads * q_pairs; i += 64) {
      const int hd = i / q_pairs, p = i % q_pairs;
      int ui, vi;
      rot_places(rot, p, &ui, &vi);
      T* src = row + hd * (a.DP + RP) + a.DP;
      float u = to_f32(src[ui]), v = to_f32(src[vi]);
      if (p < pairs) {
        const float z = u * cs[p] - v * sn[p];
        v = v * cs[p] + u * sn[p];
        u = z;
      }
      T* dst = absorbed
                   ? a.q_abs + ((long)t * a.heads + hd) * (CP + RP) + CP
                   : src;
      dst[ui] = from_f32<T>(u);
      dst[vi] = from_f32<T>(v);
    }
  }
  if (a.cq)
    wave_norm(a.cq_out + (long)t * a.QP, a.cq + (long)t * a.ld_lat, a.q_norm,
              a.QP, a.q_rank, eps);
  if (!a.lat) return;
  const T* lat = a.lat + (long)t * a.ld_lat;
  const long slot = slots[t];
  if (slot < 0 || slot >= a.n_slots) return;
  T* dst = a.cache + slot * (CP + RP);
  wave_norm(dst, lat, a.kv_norm, CP, a.kv_rank, eps);
  for (int p = lane; p < hp; p += 64) {
    int ui, vi;
    rot_places(rot, p, &ui, &vi);
    float u = to_f32(lat[CP + ui]), v = to_f32(lat[CP + vi]);
    if (p < pairs) {
      const float z = u * cs[p] - v * sn[p];
      v = v * cs[p] + u * sn[p];
      u = z;
    }
    dst[CP + ui] = from_f32<T>(u);
    dst[CP + vi] = from_f32<T>(v);
  }
}

// ------------------------------------------------------------------- //
// per-head product: out[t, h, :N] = a[t, h, :K] @ w[h]^T   (w [H, N, K])
// one wave per 16 x 16 output tile; operands straight from L2/HBM
// ------------------------------------------------------------------- //
// gate: out *= sigmoid(gate[t, h * N + n]). rot: the last workgroup of a row
// also turns a's RP elements behind K and puts them behind out's N.
template <typename T>
__global__ __launch_bounds__(256) void head_gemm_kernel(
    const T* __restrict__ a, long a_t, long a_h, const T* __restrict__ w,
    T* __restrict__ out, long o_t, long o_h, int M, int N, int K,
    const T* __restrict__ gate, long g_t, Rot rot, int RP,
    const int* __restrict__ positions) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int h = blockIdx.y;
  const int m0 = blockIdx.z * 16;
  if (RP > 0 && blockIdx.x == gridDim.x - 1) {
    const int hp = RP / 2;
    for (int i = threadIdx.x; i < 16 * hp; i += 256) {
      const int t = m0 + i / hp, p = i % hp;
      if (t >= M) break;
      int ui, vi;
      rot_places(rot, p, &ui, &vi);
      const T* src = a + (long)t * a_t + (long)h * a_h + K;
      T* dst = out + (long)t * o_t + (long)h * o_h + N;
      float u = to_f32(src[ui]), v = to_f32(src[vi]);
      if (p < rot.pairs) {
        float s, c;
        sincosf((float)positions[t] * rot.inv_freq[p], &s, &c);
        c *= rot.gain;
        s *= rot.gain;
        const float z = u * c - v * s;
        v = v * c + u * s;
        u = z;
      }
      dst[ui] = from_f32<T>(u);
      dst[vi] = from_f32<T>(v);
    }
    return;
  }
  const int n0 = (blockIdx.x * 4 + wave) * 16;
  if (n0 >= N) return;
  const int r16 = lane & 15, ko = (lane >> 4) * 8;
  const T* wr = w + ((long)h * N + n0 + r16) * K + ko;
  const T* ar = a + (long)min(m0 + r16, M - 1) * a_t + (long)h * a_h + ko;
  lm_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k = 0; k < K; k += 32)
    acc = mma32(load_frag(wr + k), load_frag(ar + k), acc);
  // C: row (n) = 4 * (lane >> 4) + r, column (token) = lane & 15
  const int m = m0 + r16, n = n0 + 4 * (lane >> 4);
  if (m < M) {
    float f[4] = {acc[0], acc[1], acc[2], acc[3]};
    if (gate) {
      const T* g = gate + (long)m * g_t + (long)h * N + n;
#pragma unroll
      for (int r = 0; r < 4; ++r) f[r] *= sigmoid_f(to_f32(g[r]));
    }
    store4(out + (long)m * o_t + (long)h * o_h + n, f);
  }
}

// ------------------------------------------------------------------- //
// absorbed attention: one token x 16 heads x one key range per workgroup
// ------------------------------------------------------------------- //
// Each wave walks 32-key tiles of its own: rows go through registers into a
// wave-private LDS tile (the next tile's loads are in flight while this one
// is multiplied), S^T = K Q^T stays in registers and is directly the second
// product's operand, o^T[c][head] += c^T p^T. No barrier until the waves'
// partial sums meet at the end. NT: 16-column latent tiles per workgroup.
template <typename T, int NT>
__global__ __launch_bounds__(256, 1) void latent_attn_kernel(
    const T* __restrict__ q_abs,  // [n, H, CP+RP]
    const T* __restrict__ cache, const int* __restrict__ block_table,
    const int* __restrict__ tok_seq, const int* __restrict__ positions,
    const T* __restrict__ sink, T* __restrict__ out,  // [n, H, CP]
    float* __restrict__ part_o, float* __restrict__ part_ml, int splits,
    int col_groups, int H, int CP, int RP, int block_size, int max_blocks,
    int n_blocks, int n_seqs, int window, float scale) {
  // bf16: the next tile's rows wait in registers, one 16-byte piece of every
  // row per lane; 32-bit tiles (exact runs) load when they are stored
  constexpr bool PRE = sizeof(T) == 2;
  const int ROW = CP + RP, PITCH = ROW + 8;
  const int nw = blockDim.x >> 6;
  extern __shared__ __align__(16) char smem[];
  __shared__ float stat[4][16][2];
  T* qs = (T*)smem;                        // [16][PITCH]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  T* tile = qs + 16 * PITCH + wave * 32 * PITCH;  // [32][PITCH]
  const int r16 = lane & 15, g = lane >> 4, ko = g * 8;
  const int t = blockIdx.x;
  const int h0 = blockIdx.y * 16;
  const int split = blockIdx.z / col_groups;
  const int c_base = (blockIdx.z % col_groups) * (NT * 16);
  const float scale2 = scale * LM_LOG2E;

  const int pos = min(max(positions[t], 0), max_blocks * block_size - 1);
  const int* btab = block_table +
                    (long)min(max(tok_seq[t], 0), n_seqs - 1) * max_blocks;
  const int lo = window > 0 ? max(0, pos - window + 1) : 0;
  const int n_tiles = (pos + 1 - lo + 31) / 32;
  const int stride = splits * nw;
  int j = split * nw + wave;

  const int row8 = ROW / 8;
  // cached row of key `lane & 31` of a tile; behind the last key, that key's
  auto row_of = [&](int jt) {
    const int key = min(lo + jt * 32 + (lane & 31), pos);
    const int blk = min(max(btab[key / block_size], 0), n_blocks - 1);
    return blk * block_size + key % block_size;
  };
  // Lane l moves columns 8l..8l+7 of each row, so that a row's address is
  // uniform; columns behind the 64th piece (rows of more than 512) go late.
  uint32x4 pre[PRE ? 32 : 1];
  const bool has_piece = lane < row8;
  auto load = [&](int rows) {
    if (PRE && has_piece) {
#pragma unroll
      for (int k = 0; k < 32; ++k) {
        const long r = __builtin_amdgcn_readlane(rows, k);
        pre[PRE ? k : 0] = *reinterpret_cast<const uint32x4*>(
            cache + r * ROW + lane * 8);
      }
    }
  };
  auto store = [&](int rows) {
    if (PRE && has_piece) {
#pragma unroll
      for (int k = 0; k < 32; ++k)
        *reinterpret_cast<uint32x4*>(tile + k * PITCH + lane * 8) =
            pre[PRE ? k : 0];
    }
    const int c0 = PRE ? 64 : 0, rest = row8 - c0;
    for (int p = lane; p < 32 * rest; p += 64) {
      const int k = p / rest, c = (c0 + p % rest) * 8;
      const long r = __shfl(rows, k, 64);
      copy8(tile + k * PITCH + c, cache + r * ROW + c);
    }
  };

  int rows = row_of(j), rows_n = row_of(j + stride);
  if (j < n_tiles) load(rows);
  for (int i = tid; i < 16 * row8; i += blockDim.x) {
    const int r = i / row8, c = (i % row8) * 8;
    if (h0 + r < H) copy8(qs + r * PITCH + c,
                          q_abs + ((long)t * H + h0 + r) * ROW + c);
    else zero8(qs + r * PITCH + c);
  }
  __syncthreads();

  float m_run = -INFINITY, l_run = 0.f;  // head r16, this lane group's keys
  lm_f32x4 acc[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) acc[i] = lm_f32x4{0.f, 0.f, 0.f, 0.f};

  for (; j < n_tiles; j += stride) {
    wave_lds_fence();  // the previous tile has been read
    store(rows);
    rows = rows_n;
    if (j + stride < n_tiles) load(rows);
    rows_n = row_of(j + 2 * stride);
    wave_lds_fence();
    lm_f32x4 s[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll 4
    for (int k = 0; k < ROW; k += 32) {
      const Frag<T> qf = load_frag(qs + r16 * PITCH + k + ko);
      s[0] = mma32(load_frag(tile + r16 * PITCH + k + ko), qf, s[0]);
      s[1] = mma32(load_frag(tile + (16 + r16) * PITCH + k + ko), qf, s[1]);
    }
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = lo + j * 32 + i * 16 + 4 * g + r;
        s[i][r] = key <= pos ? s[i][r] * scale2 : -INFINITY;
        mx = fmaxf(mx, s[i][r]);
      }
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float m_new = fmaxf(m_run, mx);  // finite: a tile has a key
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
    m_run = m_new;
    l_run *= alpha;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        s[i][r] = __builtin_amdgcn_exp2f(s[i][r] - m_new);
        l_run += s[i][r];
      }
    }
    const Frag<T> pf = frag_of<T>(s[0], s[1]);
    // columns behind CP (NT is rounded up) sum what lies there in LDS and
    // are dropped at the end
#pragma unroll
    for (int i = 0; i < NT; ++i) acc[i] *= alpha;
#pragma unroll
    for (int i = 0; i < NT; ++i)
      acc[i] = mma32(load_frag_rows(tile + c_base + i * 16, PITCH), pf,
                     acc[i]);
  }

  // the wave's own tile region holds its sums
  const int cols = min(NT * 16, CP - c_base);
  meet_waves<NT>(
      acc, m_run, l_run, cols, min(16, H - h0), stat,
      (float*)(qs + 16 * PITCH), 32 * PITCH * (int)sizeof(T) / 4,
      [&](int r, int c, const lm_f32x4& o, float m, float l) {
        const int h = h0 + r;
        if (splits > 1) {
          const long pi = ((long)t * H + h) * splits + split;
          const float v[4] = {o[0], o[1], o[2], o[3]};
          store4(part_o + pi * CP + c_base + c, v);
          if (c == 0 && c_base == 0) {
            part_ml[2 * pi] = m;
            part_ml[2 * pi + 1] = l;
          }
        } else {
          const float inv = over_weights(
              m, l, sink ? to_f32(sink[h]) * LM_LOG2E : -INFINITY);
          const float v[4] = {o[0] * inv, o[1] * inv, o[2] * inv, o[3] * inv};
          store4(out + ((long)t * H + h) * CP + c_base + c, v);
        }
      });
}

}  // namespace

// q [T, heads * (DP + RP)]; lat [T, CP + RP] with kv_norm and cache; cq
// [T, QP] (same row stride as lat) with q_norm -> returned normed rows
c10::optional<torch::Tensor> lm_latent_prep(
    c10::optional<torch::Tensor> q, c10::optional<torch::Tensor> lat,
    c10::optional<torch::Tensor> cq, torch::Tensor positions,
    torch::Tensor slots, torch::Tensor inv_freq, double gain, bool half,
    long heads, long DP, long RP, long CP, long kv_rank, double eps,
    c10::optional<torch::Tensor> kv_norm, c10::optional<torch::Tensor> cache,
    c10::optional<torch::Tensor> q_abs, long n_abs,
    c10::optional<torch::Tensor> q_norm, long q_rank) {
  LM_CHECK_I32(positions);
  LM_CHECK_I32(slots);
  const long T = positions.numel();
  TORCH_CHECK(q.has_value() || lat.has_value());
  const auto& any = q ? *q : *lat;
  const auto type = any.scalar_type();
  TORCH_CHECK(DP % 32 == 0 && RP % 32 == 0 && CP % 32 == 0);
  const Rot rot = make_rot(inv_freq, gain, half, RP);
  TORCH_CHECK(slots.numel() == T);
  TORCH_CHECK(n_abs >= 0 && n_abs <= T);
  if (q) lm_check_rows(*q, T, heads * (DP + RP), type);
  if (n_abs > 0) {
    TORCH_CHECK(q.has_value() && q_abs.has_value());
    LM_CHECK_CONTIG(*q_abs);
    TORCH_CHECK(q_abs->numel() == n_abs * heads * (CP + RP) &&
                q_abs->scalar_type() == type);
  }
  long n_slots = 0;
  if (lat) {
    lm_check_rows(*lat, T, CP + RP, type);
    TORCH_CHECK(cache.has_value() && kv_norm.has_value());
    LM_CHECK_CONTIG(*cache);
    TORCH_CHECK(cache->dim() == 3 && cache->size(2) == CP + RP &&
                cache->scalar_type() == type);
    TORCH_CHECK(kv_norm->is_contiguous() && kv_norm->numel() == CP &&
                kv_norm->scalar_type() == type && kv_rank >= 1);
    n_slots = (long)cache->size(0) * cache->size(1);
  }
  c10::optional<torch::Tensor> out;
  long QP = 0;
  if (cq) {
    QP = cq->size(1);
    TORCH_CHECK(lat.has_value() && QP % 8 == 0 && q_rank >= 1);
    lm_check_rows(*cq, T, QP, type);
    TORCH_CHECK(T <= 1 || cq->stride(0) == lat->stride(0));
    TORCH_CHECK(q_norm.has_value() && q_norm->is_contiguous() &&
                q_norm->numel() == QP && q_norm->scalar_type() == type);
    out = torch::empty({T, QP}, any.options());
  }
  if (T == 0) return out;
  LM_DISPATCH(any, "lm_latent_prep", [&] {
    PrepArgs<scalar_t> a{};
    if (q) {
      a.q = (scalar_t*)q->data_ptr();
      a.ldq = q->stride(0);
      a.heads = (int)heads;
      a.DP = (int)DP;
      a.q_abs = n_abs > 0 ? (scalar_t*)q_abs->data_ptr() : nullptr;
      a.n_abs = (int)n_abs;
    }
    if (lat) {
      a.lat = (const scalar_t*)lat->data_ptr();
      a.ld_lat = lat->stride(0);
      a.kv_norm = (const scalar_t*)kv_norm->data_ptr();
      a.kv_rank = (int)kv_rank;
      a.cache = (scalar_t*)cache->data_ptr();
      a.n_slots = n_slots;
    }
    if (cq) {
      a.cq = (const scalar_t*)cq->data_ptr();
      a.q_norm = (const scalar_t*)q_norm->data_ptr();
      a.cq_out = (scalar_t*)out->data_ptr();
      a.QP = (int)QP;
      a.q_rank = (int)q_rank;
    }
    hipLaunchKernelGGL((latent_prep_kernel<scalar_t>),
                       dim3((T + PREP_W - 1) / PREP_W), dim3(PREP_W * 64), 0,
                       cmls::current_stream(), a, positions.data_ptr<int>(),
                       slots.data_ptr<int>(), rot, (int)RP, (int)CP,
                       (float)eps, (int)T);
  });
  LM_LAUNCHED();
  return out;
}

// with positions and inv_freq: a is [M, H, K + RP] and out [M, H, N + RP],
// whose last RP elements are a's, turned
void lm_head_gemm(torch::Tensor a, torch::Tensor w, torch::Tensor out,
                  c10::optional<torch::Tensor> gate,
                  c10::optional<torch::Tensor> positions,
                  c10::optional<torch::Tensor> inv_freq, double gain,
                  bool half, long RP) {
  LM_CHECK_CUDA(a);
  LM_CHECK_CUDA(out);
  LM_CHECK_CONTIG(w);
  TORCH_CHECK(a.dim() == 3 && w.dim() == 3 && out.dim() == 3);
  const int M = a.size(0), H = a.size(1), K = w.size(2), N = w.size(1);
  TORCH_CHECK(RP >= 0 && RP % 2 == 0);
  TORCH_CHECK(w.size(0) == H && a.size(2) == K + RP);
  TORCH_CHECK(out.size(0) == M && out.size(1) == H && out.size(2) == N + RP);
  TORCH_CHECK(a.stride(2) == 1 && out.stride(2) == 1);
  TORCH_CHECK(K % 32 == 0 && N % 16 == 0, "lm_head_gemm: K % 32, N % 16");
  TORCH_CHECK(a.stride(0) % 8 == 0 && a.stride(1) % 8 == 0 &&
              out.stride(0) % 4 == 0 && out.stride(1) % 4 == 0 &&
              a.storage_offset() % 8 == 0 && out.storage_offset() % 4 == 0);
  TORCH_CHECK(a.scalar_type() == w.scalar_type() &&
              out.scalar_type() == w.scalar_type());
  Rot rot{nullptr, 0, 0, 1.f};
  if (RP > 0) {
    TORCH_CHECK(positions.has_value() && inv_freq.has_value());
    LM_CHECK_I32(*positions);
    TORCH_CHECK(positions->numel() >= M);
    rot = make_rot(*inv_freq, gain, half, RP);
  }
  if (gate) lm_check_rows(*gate, M, (long)H * N, w.scalar_type());
  if (M == 0) return;
  TORCH_CHECK((M + 15) / 16 <= 65535 && H <= 65535);
  LM_DISPATCH(w, "lm_head_gemm", [&] {
    hipLaunchKernelGGL(
        (head_gemm_kernel<scalar_t>),
        dim3((N + 63) / 64 + (RP > 0 ? 1 : 0), H, (M + 15) / 16), dim3(256),
        0, cmls::current_stream(), (const scalar_t*)a.data_ptr(), a.stride(0),
        a.stride(1), (const scalar_t*)w.data_ptr(), (scalar_t*)out.data_ptr(),
        out.stride(0), out.stride(1), M, N, K,
        gate ? (const scalar_t*)gate->data_ptr() : nullptr,
        gate ? gate->stride(0) : 0L, rot, (int)RP,
        RP > 0 ? positions->data_ptr<int>() : nullptr);
  });
  LM_LAUNCHED();
}

torch::Tensor lm_latent_attention(torch::Tensor q_abs, torch::Tensor cache,
                                  torch::Tensor block_table,
                                  torch::Tensor tok_seq,
                                  torch::Tensor positions,
                                  c10::optional<torch::Tensor> sink,
                                  double scale, long window, long CP,
                                  long max_keys) {
  LM_CHECK_CONTIG(q_abs);
  LM_CHECK_CONTIG(cache);
  LM_CHECK_I32(block_table);
  LM_CHECK_I32(tok_seq);
  LM_CHECK_I32(positions);
  TORCH_CHECK(q_abs.dim() == 3 && cache.dim() == 3 && block_table.dim() == 2);
  const int n = q_abs.size(0), H = q_abs.size(1), ROW = q_abs.size(2);
  TORCH_CHECK(cache.size(2) == ROW && CP % 32 == 0 && ROW % 32 == 0 &&
              CP > 0 && CP < ROW);
  TORCH_CHECK(tok_seq.numel() >= n && positions.numel() >= n);
  TORCH_CHECK(n == 0 || block_table.numel() > 0);
  TORCH_CHECK(cache.scalar_type() == q_abs.scalar_type());
  if (sink) {
    LM_CHECK_CONTIG(*sink);
    TORCH_CHECK(sink->numel() == H &&
                sink->scalar_type() == q_abs.scalar_type());
  }
  auto out = torch::empty({n, H, CP}, q_abs.options());
  if (n == 0) return out;
  const int hg = (H + 15) / 16;
  const int tiles = (int)(CP / 16);
  const int nt = tiles <= 2 ? 2 : tiles <= 4 ? 4 : tiles <= 6 ? 6
               : tiles <= 8 ? 8 : tiles <= 12 ? 12 : tiles <= 16 ? 16
               : tiles <= 24 ? 24 : 32;
  const int cgroups = (tiles + nt - 1) / nt;
  const int isz = q_abs.element_size();
  // the slack holds reads of rounded-up columns behind the last row
  const long slack = (long)std::max<long>(0, (long)cgroups * nt * 16 - ROW);
  auto lds = [&](int nw) {
    return ((long)(16 + 32 * nw) * (ROW + 8) + slack) * isz;
  };
  int nw = 4;
  while (nw > 1 && lds(nw) > 156 * 1024) --nw;
  TORCH_CHECK(lds(nw) <= 156 * 1024, "lm_latent_attention: kv_rank + rot_dim ",
              ROW, " does not fit LDS");
  // fill 256 CUs as far as there are 32-key tiles for every wave
  const long keys = window > 0 ? std::min(window, max_keys) : max_keys;
  const long per_cu = std::min<long>(2, 156 * 1024 / lds(nw));
  long splits = 256 * per_cu / std::max<long>(1, (long)n * hg * cgroups);
  splits = std::max<long>(1, std::min(splits,
                                      (keys + 32 * nw - 1) / (32 * nw)));
  TORCH_CHECK(hg <= 65535 && splits * cgroups <= 65535);
  torch::Tensor po, pml;
  if (splits > 1) {
    auto f32 = q_abs.options().dtype(at::kFloat);
    po = torch::empty({n, H, splits, CP}, f32);
    pml = torch::empty({n, H, splits, 2}, f32);
  }
  hipStream_t st = cmls::current_stream();
#define LM_LA(NT)                                                            \
  do {                                                                       \
    const int bytes = (int)lds(nw);                                          \
    auto* fn = &latent_attn_kernel<scalar_t, NT>;                            \
    HIP_CHECK(hipFuncSetAttribute(                                           \
        reinterpret_cast<const void*>(fn),                                   \
        hipFuncAttributeMaxDynamicSharedMemorySize, bytes));                 \
    hipLaunchKernelGGL(fn, dim3(n, hg, splits * cgroups), dim3(64 * nw),     \
                       bytes, st, (const scalar_t*)q_abs.data_ptr(),         \
                       (const scalar_t*)cache.data_ptr(),                    \
                       block_table.data_ptr<int>(), tok_seq.data_ptr<int>(), \
                       positions.data_ptr<int>(),                            \
                       sink ? (const scalar_t*)sink->data_ptr() : nullptr,   \
                       (scalar_t*)out.data_ptr(),                            \
                       splits > 1 ? po.data_ptr<float>() : nullptr,          \
                       splits > 1 ? pml.data_ptr<float>() : nullptr,         \
                       (int)splits, cgroups, H, (int)CP, (int)(ROW - CP),    \
                       (int)cache.size(1), (int)block_table.size(1),         \
                       (int)cache.size(0), (int)block_table.size(0),         \
                       (int)window, (float)scale);                           \
  } while (0)
  LM_DISPATCH(q_abs, "lm_latent_attention", [&] {
    switch (nt) {
      case 2: LM_LA(2); break;
      case 4: LM_LA(4); break;
      case 6: LM_LA(6); break;
      case 8: LM_LA(8); break;
      case 12: LM_LA(12); break;
      case 16: LM_LA(16); break;
      case 24: LM_LA(24); break;
      default: LM_LA(32); break;
    }
    if (splits > 1)
      hipLaunchKernelGGL((combine_ranges_kernel<scalar_t>), dim3(n * H),
                         dim3(128), 0, st, po.data_ptr<float>(),
                         pml.data_ptr<float>(),
                         sink ? (const scalar_t*)sink->data_ptr() : nullptr,
                         (scalar_t*)out.data_ptr(), H * CP, (int)splits, H,
                         (int)CP, 1.f);
  });
#undef LM_LA
  LM_LAUNCHED();
  return out;
}
