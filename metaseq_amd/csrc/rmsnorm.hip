// RMS norms of hybrid decoders with what surrounds them fused in: the embedding with sinusoidal
// positions, the tail of a sublayer (split-K sums, the combination of routed experts, post-norm,
// residual add, next pre-norm), the latent norms with the cache append, and small row utilities.
// One workgroup per token; a row lives in registers (NV float4 per thread): 256 threads where there
// are many tokens, up to 1024 where there are few and the latency of one row counts.
#include <math.h>

#include "common.h"

namespace {

constexpr int RN_THREADS = 256;       // latent norms; norms of many rows
constexpr int RN_FEW_ROWS = 1024;     // up to here a row is spread over more threads

// one activation element group: 4 consecutive columns of row m
template <typename T>
__device__ __forceinline__ void store_act4(void* h, int64_t m, int64_t ld, int mb, int c, float4_t v) {
  if constexpr (sizeof(T) == 4) {
    *reinterpret_cast<float4_t*>((float*)h + m * ld + c) = v;
  } else {
    bf16_t* p = (bf16_t*)h + (mb > 0 ? packed_act_offset((int)m, c, mb) : m * ld + c);
    *reinterpret_cast<bf16x4_t*>(p) = bf16x4_t{(bf16_t)v[0], (bf16_t)v[1], (bf16_t)v[2], (bf16_t)v[3]};
  }
}

__device__ __forceinline__ float dot4(float4_t v) {
  return v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
}

// x (registers) -> h = x / rms(x) * w
template <typename T, int NV, int NT>
__device__ __forceinline__ void norm_out(const float4_t (&x)[NV], int64_t m, int D, int Dp, float eps,
                                         const float* w, void* h, int mb, float* red) {
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) ss += dot4(x[i]);
  ss = block_sum(ss, red);
  const float r = 1.f / sqrtf(ss / (float)D + eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + i * NT) * 4;
    if (c < Dp) {
      const float4_t wv = *reinterpret_cast<const float4_t*>(w + c);
      store_act4<T>(h, m, Dp, mb, c, x[i] * r * wv);
    }
  }
}

template <typename T, int NV, int NT>
__global__ __launch_bounds__(NT) void embed_kernel(
    const int64_t* __restrict__ tokens, const int32_t* __restrict__ tok_pos,
    const bf16_t* __restrict__ table, int vocab, float scale, const double* __restrict__ inv_freq,
    int D, int Dp, float eps, const float* __restrict__ step, float* __restrict__ e_out,
    float* __restrict__ x, const float* __restrict__ w, void* h, int mb) {
  __shared__ float red[16];
  const int64_t m = blockIdx.x;
  int64_t t = tokens[m];
  t = t < 0 ? 0 : (t >= vocab ? vocab - 1 : t);
  const double pos = (double)max(tok_pos[m], 0);
  float4_t v[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + i * NT) * 4;
    v[i] = float4_t{0.f, 0.f, 0.f, 0.f};
    if (c >= Dp) continue;
    const bf16x4_t e = *reinterpret_cast<const bf16x4_t*>(table + t * Dp + c);
#pragma unroll
    for (int j = 0; j < 4; j += 2) {
      float sn = 0.f, cs = 0.f;
      if (inv_freq && c + j < D) {
        // the angle in turns, reduced to [-1/2, 1/2] in double; sine and cosine of pi * (2 turns)
        double turns = pos * inv_freq[(c + j) >> 1] * 0.15915494309189535;
        turns -= rint(turns);
        sincospif(2.f * (float)turns, &sn, &cs);
      }
      v[i][j] = (float)e[j] * scale + sn;
      v[i][j + 1] = (float)e[j + 1] * scale + (c + j + 1 < D ? cs : 0.f);
    }
    if (e_out) *reinterpret_cast<float4_t*>(e_out + m * Dp + c) = v[i];
    if (step) v[i] += *reinterpret_cast<const float4_t*>(step + c);
    *reinterpret_cast<float4_t*>(x + m * Dp + c) = v[i];
  }
  if (w) norm_out<T, NV, NT>(v, m, D, Dp, eps, w, h, mb, red);
}

// b += the sum of S slices of row m; four slices at a time, their loads in flight together
template <int NV, int NT>
__device__ __forceinline__ void sum_slices(const float* part, int S, int M, int64_t m, int Dp,
                                           float4_t (&b)[NV]) {
  for (int s0 = 0; s0 < S; s0 += 4) {
    float4_t v[4][NV];
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const float* p = part + ((int64_t)min(s0 + s, S - 1) * M + m) * Dp;
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int c = (threadIdx.x + i * NT) * 4;
        v[s][i] = c < Dp && s0 + s < S ? *reinterpret_cast<const float4_t*>(p + c)
                                       : float4_t{0.f, 0.f, 0.f, 0.f};
      }
    }
#pragma unroll
    for (int s = 0; s < 4; ++s)
#pragma unroll
      for (int i = 0; i < NV; ++i) b[i] += v[s][i];
  }
}

// TWO: a second sublayer beside the first (part2)
template <typename T, int NV, int NT, bool TWO>
__global__ __launch_bounds__(NT) void tail_kernel(msa_tail_args a) {
  __shared__ float red[32];
  const int64_t m = blockIdx.x;
  const int D = a.D, Dp = a.Dp;
  float4_t b[NV], x[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + i * NT) * 4;
    b[i] = x[i] = float4_t{0.f, 0.f, 0.f, 0.f};
    if (c < Dp) x[i] = *reinterpret_cast<const float4_t*>(a.x + m * Dp + c);
  }
  if (a.part) {
    sum_slices<NV, NT>(a.part, a.S, a.M, m, Dp, b);
    if (a.gate) {
      const float g = a.gate[m];
#pragma unroll
      for (int i = 0; i < NV; ++i) b[i] = b[i] * g;
    }
    if (a.bias) {
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int c = (threadIdx.x + i * NT) * 4;
        if (c < Dp) b[i] += *reinterpret_cast<const float4_t*>(a.bias + c);
      }
    }
  }
  if (a.pair_y) {
    typedef T t4 __attribute__((ext_vector_type(4)));
    constexpr int U = NV <= 2 ? 4 : 1;
    for (int k0 = 0; k0 < a.top; k0 += U) {
      t4 y[U][NV];
      float w[U];
#pragma unroll
      for (int k = 0; k < U; ++k) {
        const int64_t at = m * a.top + min(k0 + k, a.top - 1);
        w[k] = k0 + k < a.top ? a.pair_w[at] : 0.f;
        const T* p = (const T*)a.pair_y + (int64_t)a.inverse[at] * Dp;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
          const int c = (threadIdx.x + i * NT) * 4;
          y[k][i] = *reinterpret_cast<const t4*>(p + (c < Dp ? c : 0));
        }
      }
#pragma unroll
      for (int k = 0; k < U; ++k)
        if (k0 + k < a.top) {  // uniform
#pragma unroll
          for (int i = 0; i < NV; ++i)
#pragma unroll
            for (int j = 0; j < 4; ++j) b[i][j] += w[k] * (float)y[k][i][j];
        }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if ((threadIdx.x + i * NT) * 4 >= Dp) b[i] = float4_t{0.f, 0.f, 0.f, 0.f};
  }
  float r = 1.f;
  if constexpr (TWO) {
    float4_t b2[NV];
    float ss = 0.f, ss2 = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) b2[i] = float4_t{0.f, 0.f, 0.f, 0.f};
    sum_slices<NV, NT>(a.part2, a.S2, a.M, m, Dp, b2);
#pragma unroll
    for (int i = 0; i < NV; ++i) ss += dot4(b[i]), ss2 += dot4(b2[i]);
    block_sum2(ss, ss2, red);
    r = 1.f / sqrtf(ss / (float)D + a.eps);
    const float r2 = 1.f / sqrtf(ss2 / (float)D + a.eps);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (threadIdx.x + i * NT) * 4;
      if (c < Dp) x[i] += b2[i] * r2 * *reinterpret_cast<const float4_t*>(a.w_post2 + c);
    }
  } else if (a.w_post) {
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) ss += dot4(b[i]);
    ss = block_sum(ss, red);
    r = 1.f / sqrtf(ss / (float)D + a.eps);
  }
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (threadIdx.x + i * NT) * 4;
    if (c < Dp) {
      if (a.w_post) {
        const float4_t wv = *reinterpret_cast<const float4_t*>(a.w_post + c);
        b[i] = b[i] * r * wv;
      }
      x[i] += b[i];
      if (a.probe) *reinterpret_cast<float4_t*>(a.probe + m * Dp + c) = x[i];
      if (a.add) x[i] += *reinterpret_cast<const float4_t*>(a.add + m * Dp + c);
      if (a.step) x[i] += *reinterpret_cast<const float4_t*>(a.step + c);
      *reinterpret_cast<float4_t*>(a.x + m * Dp + c) = x[i];
    }
  }
  if (a.w_next) norm_out<T, NV, NT>(x, m, D, Dp, a.eps, a.w_next, a.h, a.h_mb, red);
}

// Down-projected latents: one workgroup per token, the two norms by different halves of it.
template <typename T>
__global__ __launch_bounds__(RN_THREADS) void latent_norm_kernel(
    const float* __restrict__ part, int S, int N, int M, int q_rank, int qp,
    const float* __restrict__ wq, int kv_rank, int rp, const float* __restrict__ wkv, float eps,
    void* cq, int cq_mb, T* latent, int capacity, const int32_t* __restrict__ tok_slot,
    const int32_t* __restrict__ tok_pos) {
  __shared__ float red[16];
  __shared__ float row[4096];  // summed latents of this token (N <= 4096)
  const int64_t m = blockIdx.x;
  float sq = 0.f, skv = 0.f;
  for (int c = threadIdx.x; c < qp + rp; c += RN_THREADS) {
    float v = 0.f;
    for (int s0 = 0; s0 < S; s0 += 4) {
      float p[4];
#pragma unroll
      for (int s = 0; s < 4; ++s)
        p[s] = s0 + s < S ? part[((int64_t)min(s0 + s, S - 1) * M + m) * N + c] : 0.f;
      v += (p[0] + p[1]) + (p[2] + p[3]);
    }
    row[c] = v;
    if (c < qp) sq += v * v;
    else skv += v * v;
  }
  sq = block_sum(sq, red);
  const float rq = 1.f / sqrtf(sq / (float)q_rank + eps);
  for (int c = threadIdx.x * 4; c < qp; c += RN_THREADS * 4) {
    const float4_t v = *reinterpret_cast<const float4_t*>(row + c);
    store_act4<T>(cq, m, qp, cq_mb, c, v * rq * *reinterpret_cast<const float4_t*>(wq + c));
  }
  if (!latent) return;
  skv = block_sum(skv, red);
  const float rkv = 1.f / sqrtf(skv / (float)kv_rank + eps);
  const int pos = tok_pos[m];
  if (pos < 0 || pos >= capacity) return;
  T* dst = latent + ((int64_t)tok_slot[m] * capacity + pos) * rp;
  for (int c = threadIdx.x * 4; c < rp; c += RN_THREADS * 4) {
    const float4_t v = *reinterpret_cast<const float4_t*>(row + qp + c);
    store_act4<T>(dst, 0, rp, 0, c, v * rkv * *reinterpret_cast<const float4_t*>(wkv + c));
  }
}

template <typename T>
__global__ void zero_columns_kernel(T* y, int64_t M, int64_t ld, int mb, int c0, int c1) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  const int w = c1 - c0;
  if (i >= M * w) return;
  const int64_t m = i / w;
  const int c = c0 + (int)(i - m * w);
  y[mb > 0 ? packed_act_offset((int)m, c, mb) : m * ld + c] = (T)0.f;
}

// 8 elements (16 or 32 bytes) per thread; rows past n of a packed destination stay as they are
template <typename T>
__global__ void gather_rows_kernel(const T* src, int src_mb, const int32_t* rows, int n, int K, T* dst,
                                   int dst_mb) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  const int q = K / 8;
  if (i >= (int64_t)n * q) return;
  const int r = (int)(i / q), c = (int)(i % q) * 8;
  const int64_t m = rows[r];
  typedef T t8 __attribute__((ext_vector_type(8), aligned(16)));
  const T* s = src + (src_mb > 0 ? packed_act_offset((int)m, c, src_mb) : m * K + c);
  T* d = dst + (dst_mb > 0 ? packed_act_offset(r, c, dst_mb) : (int64_t)r * K + c);
  *reinterpret_cast<t8*>(d) = *reinterpret_cast<const t8*>(s);
}

__global__ void step_positions_kernel(const int32_t* lens, const int64_t* tokens, int64_t stride,
                                      int64_t pad, int B, int32_t* step_pos) {
  const int b = blockIdx.x * 256 + threadIdx.x;
  if (b < B) step_pos[b] = lens[b] >= 0 && tokens[b * stride] != pad ? lens[b] : -1;
}

__global__ void advance_active_kernel(int32_t* lens, const int32_t* step_pos, int B) {
  const int b = blockIdx.x * 256 + threadIdx.x;
  if (b < B && step_pos[b] >= 0) lens[b] = step_pos[b] + 1;
}

constexpr int RN_MAX_WIDTH = 16384;

// one row per workgroup of NT threads with NV float4 each
#define RN_RUN(KERNEL, T, NV, NT, M, ...) \
  hipLaunchKernelGGL((KERNEL<T, NV, NT>), dim3(M), dim3(NT), 0, (hipStream_t)stream, __VA_ARGS__)
template <typename T, int NV, int NT>
constexpr auto tail_one = tail_kernel<T, NV, NT, false>;
template <typename T, int NV, int NT>
constexpr auto tail_two = tail_kernel<T, NV, NT, true>;
#define RN_DISPATCH(KERNEL, T, M, Dp, ...)                                                  \
  do {                                                                                      \
    const int q_ = (Dp) / 4;                                                                \
    if (q_ <= 256) RN_RUN(KERNEL, T, 1, 256, M, __VA_ARGS__);                               \
    else if ((M) <= RN_FEW_ROWS) {                                                          \
      if (q_ <= 512) RN_RUN(KERNEL, T, 1, 512, M, __VA_ARGS__);                             \
      else if (q_ <= 1024) RN_RUN(KERNEL, T, 1, 1024, M, __VA_ARGS__);                      \
      else if (q_ <= 2048) RN_RUN(KERNEL, T, 2, 1024, M, __VA_ARGS__);                      \
      else RN_RUN(KERNEL, T, 4, 1024, M, __VA_ARGS__);                                      \
    } else if (q_ <= 512) RN_RUN(KERNEL, T, 2, 256, M, __VA_ARGS__);                        \
    else if (q_ <= 1024) RN_RUN(KERNEL, T, 4, 256, M, __VA_ARGS__);                         \
    else if (q_ <= 2048) RN_RUN(KERNEL, T, 4, 512, M, __VA_ARGS__);                         \
    else RN_RUN(KERNEL, T, 4, 1024, M, __VA_ARGS__);                                        \
  } while (0)

}  // namespace

extern "C" int msa_embed_rmsnorm(int dtype, const int64_t* tokens, const int32_t* tok_pos, int M,
                                 const void* table, int vocab, float scale, const double* inv_freq,
                                 int D, int Dp, float eps, const float* step, float* e, float* x,
                                 const float* w, void* h, int h_mb, void* stream) {
  const char* name = "msa_embed_rmsnorm";
  MSA_REQUIRE(tokens && tok_pos && table && x && (!w || h), MSA_ERR_INVALID_ARG,
              "%s: null pointer", name);
  MSA_REQUIRE(M > 0 && vocab > 0 && D > 0 && D <= Dp && Dp % 4 == 0 && Dp <= RN_MAX_WIDTH, MSA_ERR_INVALID_ARG,
              "%s: M=%d vocab=%d D=%d Dp=%d", name, M, vocab, D, Dp);
  if (dtype == MSA_BF16)
    RN_DISPATCH(embed_kernel, bf16_t, M, Dp, tokens,
                tok_pos, (const bf16_t*)table, vocab, scale, inv_freq, D, Dp, eps, step, e, x, w, h,
                h_mb);
  else
    RN_DISPATCH(embed_kernel, float, M, Dp, tokens,
                tok_pos, (const bf16_t*)table, vocab, scale, inv_freq, D, Dp, eps, step, e, x, w, h, 0);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_residual_rmsnorm_tail(const msa_tail_args* a, void* stream) {
  const char* name = "msa_residual_rmsnorm_tail";
  MSA_REQUIRE(a && a->x && (a->part || a->pair_y) && (!a->w_next || a->h), MSA_ERR_INVALID_ARG,
              "%s: null pointer", name);
  MSA_REQUIRE(!a->pair_y || (a->pair_w && a->inverse && a->top > 0), MSA_ERR_INVALID_ARG,
              "%s: routed terms without weights", name);
  MSA_REQUIRE(a->M > 0 && a->D > 0 && a->D <= a->Dp && a->Dp % 4 == 0 && a->Dp <= RN_MAX_WIDTH &&
                  (!a->part || a->S > 0),
              MSA_ERR_INVALID_ARG, "%s: M=%d D=%d Dp=%d S=%d", name, a->M, a->D, a->Dp, a->S);
  MSA_REQUIRE(!a->part2 || (a->part && a->w_post && a->w_post2 && a->S2 > 0), MSA_ERR_INVALID_ARG,
              "%s: a second sublayer beside none, or without norms", name);
  MSA_REQUIRE(!a->bias || a->part, MSA_ERR_INVALID_ARG, "%s: a bias without a product", name);
  if (a->part2) {
    if (a->dtype == MSA_BF16)
      RN_DISPATCH(tail_two, bf16_t, a->M, a->Dp, *a);
    else
      RN_DISPATCH(tail_two, float, a->M, a->Dp, *a);
  } else if (a->dtype == MSA_BF16) {
    RN_DISPATCH(tail_one, bf16_t, a->M, a->Dp, *a);
  } else {
    RN_DISPATCH(tail_one, float, a->M, a->Dp, *a);
  }
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_latent_norm(int dtype, const float* part, int S, int N, int M, int q_rank, int qp,
                               const float* wq, int kv_rank, int rp, const float* wkv, float eps,
                               void* cq, int cq_mb, void* latent, int capacity, const msa_batch* b,
                               void* stream) {
  const char* name = "msa_latent_norm";
  MSA_REQUIRE(part && wq && cq && b && (!latent || wkv), MSA_ERR_INVALID_ARG, "%s: null pointer",
              name);
  const int r = latent ? rp : 0;
  MSA_REQUIRE(M > 0 && S > 0 && qp % 4 == 0 && r % 4 == 0 && qp + r <= N && qp + r <= 4096,
              MSA_ERR_INVALID_ARG, "%s: M=%d S=%d N=%d, latents of %d and %d (at most 4096 together)",
              name, M, S, N, qp, r);
  if (dtype == MSA_BF16)
    hipLaunchKernelGGL(latent_norm_kernel<bf16_t>, dim3(M), dim3(RN_THREADS), 0, (hipStream_t)stream,
                       part, S, N, M, q_rank, qp, wq, kv_rank, r, wkv, eps, cq, cq_mb,
                       (bf16_t*)latent, capacity, b->tok_slot, b->tok_pos);
  else
    hipLaunchKernelGGL(latent_norm_kernel<float>, dim3(M), dim3(RN_THREADS), 0, (hipStream_t)stream,
                       part, S, N, M, q_rank, qp, wq, kv_rank, r, wkv, eps, cq, 0, (float*)latent,
                       capacity, b->tok_slot, b->tok_pos);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_zero_columns(int dtype, void* y, int64_t M, int64_t ld, int mb, int c0, int c1,
                                void* stream) {
  MSA_REQUIRE(y && M >= 0 && c0 >= 0 && c1 <= ld, MSA_ERR_INVALID_ARG, "msa_zero_columns: bad range");
  if (M == 0 || c1 <= c0) return MSA_OK;
  const dim3 grid((unsigned)((M * (c1 - c0) + 255) / 256));
  if (dtype == MSA_BF16)
    hipLaunchKernelGGL(zero_columns_kernel<bf16_t>, grid, dim3(256), 0, (hipStream_t)stream,
                       (bf16_t*)y, M, ld, mb, c0, c1);
  else
    hipLaunchKernelGGL(zero_columns_kernel<float>, grid, dim3(256), 0, (hipStream_t)stream, (float*)y,
                       M, ld, 0, c0, c1);
  MSA_CHECK_LAUNCH("msa_zero_columns");
  return MSA_OK;
}

extern "C" int msa_gather_rows(int dtype, const void* src, int src_mb, const int32_t* rows, int n, int K,
                               void* dst, int dst_mb, void* stream) {
  MSA_REQUIRE(src && rows && dst && n >= 0 && K > 0 && K % 8 == 0, MSA_ERR_INVALID_ARG,
              "msa_gather_rows: bad arguments");
  if (n == 0) return MSA_OK;
  const dim3 grid((unsigned)(((int64_t)n * (K / 8) + 255) / 256));
  if (dtype == MSA_BF16)
    hipLaunchKernelGGL(gather_rows_kernel<bf16_t>, grid, dim3(256), 0, (hipStream_t)stream,
                       (const bf16_t*)src, src_mb, rows, n, K, (bf16_t*)dst, dst_mb);
  else
    hipLaunchKernelGGL(gather_rows_kernel<float>, grid, dim3(256), 0, (hipStream_t)stream,
                       (const float*)src, 0, rows, n, K, (float*)dst, 0);
  MSA_CHECK_LAUNCH("msa_gather_rows");
  return MSA_OK;
}

extern "C" int msa_step_positions(const int32_t* lens, const int64_t* tokens, int64_t tok_stride,
                                  int64_t pad, int B, int32_t* step_pos, void* stream) {
  MSA_REQUIRE(lens && tokens && step_pos && B > 0, MSA_ERR_INVALID_ARG,
              "msa_step_positions: bad arguments");
  hipLaunchKernelGGL(step_positions_kernel, dim3((B + 255) / 256), dim3(256), 0, (hipStream_t)stream,
                     lens, tokens, tok_stride, pad, B, step_pos);
  MSA_CHECK_LAUNCH("msa_step_positions");
  return MSA_OK;
}

extern "C" int msa_advance_active(int32_t* lens, const int32_t* step_pos, int B, void* stream) {
  MSA_REQUIRE(lens && step_pos && B > 0, MSA_ERR_INVALID_ARG, "msa_advance_active: bad arguments");
  hipLaunchKernelGGL(advance_active_kernel, dim3((B + 255) / 256), dim3(256), 0, (hipStream_t)stream,
                     lens, step_pos, B);
  MSA_CHECK_LAUNCH("msa_advance_active");
  return MSA_OK;
}
