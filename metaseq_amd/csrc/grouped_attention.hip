// Causal softmax attention of several query heads per key/value head, with rotary positions on part of
// a head, within chunks of positions counted from the sequence's start, and with a gate per head.
//
//  * What a slot keeps is one chunk: position p lies at row p - (start of p's chunk).  A step's own keys
//    and values are read from the step's rows and appended afterwards, so a portion may run over
//    several chunks and overwrite the one that its first tokens still needed.
//  * One new token per sequence (decode): the heads of a group are the columns of the MFMA tiles, a
//    wave owns 32 keys at a time straight from memory, and the four waves of a workgroup (and its
//    splits) merge their sums at the end.  Rotation and appending are part of it.  Bound: the keys and
//    values from HBM, once per 16 heads.
//  * Several: 128 queries of one head per workgroup over key tiles of 64, one pass (see
//    flash_attention_kernel, which this follows, in latent_attention.hip).
//  * fp32, and heads of more than 256: one workgroup per (token, head) on the vector ALU.
#include <math.h>

#include "attention_tiles.h"

namespace {

constexpr int GA_MAX_HEAD = 1024;

__device__ __forceinline__ int chunk_start(int pos, int chunk) {
  return chunk > 0 ? pos - pos % chunk : 0;
}

__device__ __forceinline__ float head_gate(const msa_grouped_args& a, int64_t m, int h) {
  return a.gate ? sigmoidf(a.gate[m * a.ld_gate + h]) : 1.f;
}

template <typename T>
struct Vec8 {
  typedef T type __attribute__((ext_vector_type(8), aligned(16)));
};

// sine and cosine of pos * inv_freq; the angle in turns, reduced to [-1/2, 1/2] in double
__device__ __forceinline__ void rotary_angle(int pos, double inv_freq, float& s, float& c) {
  double turns = (double)pos * inv_freq * 0.15915494309189535;
  turns -= rint(turns);
  sincospif(2.f * (float)turns, &s, &c);
}

// ---- rotary positions, appending ---------------------------------------------------------------
// One workgroup per token; V pairs of a head per thread.
template <typename T, int V>
__global__ __launch_bounds__(256) void rotate_kernel(msa_grouped_args a,
                                                     const int32_t* __restrict__ tok_slot,
                                                     const int32_t* __restrict__ tok_pos, int append) {
  __shared__ float cs[GA_MAX_HEAD / 2], sn[GA_MAX_HEAD / 2];
  const int64_t m = blockIdx.x;
  const int pos = tok_pos[m], tid = threadIdx.x, half = a.rot_dims / 2;
  if (pos < 0) return;
  T* q = (T*)a.q + m * a.ld;
  T* k = (T*)a.k + m * a.ld;
  if (half > 0) {
    for (int i = tid; i < half; i += 256) rotary_angle(pos, a.inv_freq[i], sn[i], cs[i]);
    __syncthreads();
    typedef T tv __attribute__((ext_vector_type(V), aligned(V * sizeof(T) < 16 ? V * sizeof(T) : 16)));
    const int per = half / V, total = (a.heads + a.kv_heads) * per;
    for (int e = tid; e < total; e += 256) {
      const int h = e / per, i = (e - h * per) * V;
      T* p = (h < a.heads ? q + h * a.hd : k + (h - a.heads) * a.hd) + i;
      tv u = *reinterpret_cast<const tv*>(p), v = *reinterpret_cast<const tv*>(p + half);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        const float x = (float)u[j], y = (float)v[j], c = cs[i + j], s = sn[i + j];
        u[j] = (T)(x * c - y * s);
        v[j] = (T)(y * c + x * s);
      }
      *reinterpret_cast<tv*>(p) = u;
      *reinterpret_cast<tv*>(p + half) = v;
    }
  }
  if (!append) return;
  __syncthreads();  // the keys are read back rotated
  const int row = pos - chunk_start(pos, a.chunk);
  if (row >= a.rows) return;
  typedef typename Vec8<T>::type v8;
  const T* v = (const T*)a.v + m * a.ld;
  const int kc = a.hd / 8, vc = a.vd / 8;
  const int64_t slot = (int64_t)tok_slot[m] * a.kv_heads;
  for (int e = tid; e < a.kv_heads * (kc + vc); e += 256) {
    const int g = e / (kc + vc), c = e - g * (kc + vc);
    if (c < kc)
      *reinterpret_cast<v8*>((T*)a.k_cache + ((slot + g) * a.rows + row) * a.hd + c * 8) =
          *reinterpret_cast<const v8*>(k + g * a.hd + c * 8);
    else
      *reinterpret_cast<v8*>((T*)a.v_cache + ((slot + g) * a.rows + row) * a.vd + (c - kc) * 8) =
          *reinterpret_cast<const v8*>(v + g * a.vd + (c - kc) * 8);
  }
}

constexpr int AP_TOK = 4;  // tokens per workgroup

template <typename T>
__global__ __launch_bounds__(256) void append_kernel(msa_grouped_args a,
                                                     const int32_t* __restrict__ seg_start,
                                                     const int32_t* __restrict__ seg_slot,
                                                     const int32_t* __restrict__ seg_pos) {
  typedef typename Vec8<T>::type v8;
  const int s = blockIdx.y, pos0 = seg_pos[s];
  if (pos0 < 0) return;
  const int first = seg_start[s], n = seg_start[s + 1] - first;
  const int c0 = chunk_start(pos0 + n - 1, a.chunk);  // the chunk that stays
  const int t0 = max(0, c0 - pos0) + blockIdx.x * AP_TOK, nt = min(AP_TOK, n - t0);
  const int kc = a.hd / 8, vc = a.vd / 8, per = a.kv_heads * (kc + vc);
  const int64_t slot = (int64_t)seg_slot[s] * a.kv_heads;
  for (int e = threadIdx.x; e < nt * per; e += 256) {
    const int t = e / per, g = (e - t * per) / (kc + vc), c = (e - t * per) - g * (kc + vc);
    const int row = pos0 + t0 + t - c0;
    if (row >= a.rows) continue;
    const int64_t m = (int64_t)(first + t0 + t) * a.ld;
    if (c < kc)
      *reinterpret_cast<v8*>((T*)a.k_cache + ((slot + g) * a.rows + row) * a.hd + c * 8) =
          *reinterpret_cast<const v8*>((const T*)a.k + m + g * a.hd + c * 8);
    else
      *reinterpret_cast<v8*>((T*)a.v_cache + ((slot + g) * a.rows + row) * a.vd + (c - kc) * 8) =
          *reinterpret_cast<const v8*>((const T*)a.v + m + g * a.vd + (c - kc) * 8);
  }
}

// ---- one new token per sequence, bf16 -----------------------------------------------------------
template <int VD>
constexpr int gd_pitch = VD * 2 + 16;
template <int HD>
constexpr int gd_row = HD + 8;  // elements between two staged heads
template <int HD, int VD>
constexpr int gd_lds_bytes = 4 * 32 * gd_pitch<VD> + 17 * gd_row<HD> * 2;

// FUSED: q and k come as the projection left them; the workgroup rotates its heads, and the first
// of a group's workgroups appends.
template <int HD, int VD, bool FUSED>
__global__ __launch_bounds__(256) void grouped_decode_kernel(msa_grouped_args a, int r0, int M,
                                                             const int32_t* __restrict__ tok_slot,
                                                             const int32_t* __restrict__ tok_pos,
                                                             float scale_log2) {
  constexpr int KS = HD / 32, DW = VD / 16, PITCH = gd_pitch<VD>, CH = VD / 8, VL = 32 * CH / 64;
  constexpr int ROW = gd_row<HD>, QCH = HD / 8, QL = (17 * QCH + 255) / 256;
  extern __shared__ __attribute__((aligned(16))) char lds[];  // per wave: values of 32 keys; sums
  __shared__ float sm[4][16], sl[4][16], cs[HD / 2], sn[HD / 2];
  bf16_t* lq = reinterpret_cast<bf16_t*>(lds + 4 * 32 * PITCH);  // 16 heads, the own key
  const int per = a.heads / a.kv_heads, HB = (per + 15) / 16;
  int idx = blockIdx.x;
  const int split = idx % a.splits;
  idx /= a.splits;
  const int hb = idx % HB;
  idx /= HB;
  const int g = idx % a.kv_heads, mr = idx / a.kv_heads;
  if (mr >= M) return;
  const int64_t m = r0 + mr;
  const int tid = threadIdx.x, lane = tid & 63, hc = lane & 15, lg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const bf16_t* own_k = (const bf16_t*)a.k + m * a.ld + g * HD;
  const bf16_t* own_v = (const bf16_t*)a.v + m * a.ld + g * VD;
  half8_t qr[QL];  // the heads' and the own key's elements on their way to LDS
#pragma unroll
  for (int i = 0; i < QL; ++i) {
    const int e = min(tid + 256 * i, 17 * QCH - 1), r = e / QCH;
    const bf16_t* p = r == 16 ? own_k
                              : (const bf16_t*)a.q + m * a.ld + (g * per + min(hb * 16 + r, per - 1)) * HD;
    qr[i] = *reinterpret_cast<const half8_t*>(p + (e % QCH) * 8);
  }
  const int pos = tok_pos[m];
  const int n_keys = pos < 0 ? 0 : pos - chunk_start(pos, a.chunk);  // in the cache
  const int len = split_keys(n_keys, a.splits);
  const int k_begin = split * len, k_end = min(n_keys, k_begin + len);
  const int64_t slot = (int64_t)tok_slot[m] * a.kv_heads + g;
  bf16_t* kc = (bf16_t*)a.k_cache + slot * a.rows * HD;
  bf16_t* vc = (bf16_t*)a.v_cache + slot * a.rows * VD;

  struct Tile {
    bf16x8_t k[2][KS];
    half8_t v[VL];
  } t0, t1;
  auto fetch = [&](Tile& t, int base) {
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      const bf16_t* p = kc + (int64_t)min(base + 16 * b + hc, n_keys - 1) * HD + lg * 8;
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) t.k[b][ks] = *reinterpret_cast<const bf16x8_t*>(p + ks * 32);
    }
#pragma unroll
    for (int j = 0; j < VL; ++j) {
      const int c = lane + 64 * j;
      t.v[j] = __builtin_nontemporal_load(reinterpret_cast<const half8_t*>(
          vc + (int64_t)min(base + c / CH, n_keys - 1) * VD + (c % CH) * 8));
    }
  };
  int base = k_begin + 32 * wave;  // the wave's tiles are 128 keys apart
#pragma unroll
  for (int i = 0; i < QL; ++i)
    if (tid + 256 * i < 17 * QCH)
      *reinterpret_cast<half8_t*>(lq + (tid + 256 * i) / QCH * ROW + (tid + 256 * i) % QCH * 8) = qr[i];
  if (base < k_end) {
    fetch(t0, base);
    fetch(t1, base + 128);  // past the end: the last key again
  }
  if constexpr (FUSED) {
    const int half = a.rot_dims / 2;
    for (int i = tid; i < half; i += 256) rotary_angle(pos, a.inv_freq[i], sn[i], cs[i]);
    lds_barrier();
    for (int e = tid; e < 17 * half; e += 256) {
      const int r = e / half, i = e - r * half;
      bf16_t* p = lq + r * ROW + i;
      const float x = (float)p[0], y = (float)p[half];
      p[0] = (bf16_t)(x * cs[i] - y * sn[i]);
      p[half] = (bf16_t)(y * cs[i] + x * sn[i]);
    }
  }
  lds_barrier();
  bf16x8_t qf[KS];
#pragma unroll
  for (int ks = 0; ks < KS; ++ks)
    qf[ks] = *reinterpret_cast<const bf16x8_t*>(lq + hc * ROW + ks * 32 + lg * 8);
  if (FUSED && split == 0 && hb == 0 && pos >= 0 && n_keys < a.rows) {
    for (int e = tid; e < QCH + CH; e += 256)
      if (e < QCH)
        *reinterpret_cast<half8_t*>(kc + (int64_t)n_keys * HD + e * 8) =
            *reinterpret_cast<const half8_t*>(lq + 16 * ROW + e * 8);
      else
        *reinterpret_cast<half8_t*>(vc + (int64_t)n_keys * VD + (e - QCH) * 8) =
            *reinterpret_cast<const half8_t*>(own_v + (e - QCH) * 8);
  }
  float4_t o[DW];
#pragma unroll
  for (int d = 0; d < DW; ++d) o[d] = float4_t{0.f, 0.f, 0.f, 0.f};
  float mx = -INFINITY, l = 0.f;
  if (split == 0 && wave == 0 && pos >= 0) {  // the token's own key, which every head sees
    float s = 0.f;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const bf16x8_t k = *reinterpret_cast<const bf16x8_t*>(lq + 16 * ROW + ks * 32 + lg * 8);
#pragma unroll
      for (int i = 0; i < 8; ++i) s = fmaf((float)k[i], (float)qf[ks][i], s);
    }
    s += __shfl_xor(s, 16, MSA_WAVE);
    s += __shfl_xor(s, 32, MSA_WAVE);
    mx = s * scale_log2;
    l = lg == 0 ? 1.f : 0.f;  // the lane groups are summed at the end
#pragma unroll
    for (int d = 0; d < DW; ++d) {
      const bf16x4_t v = *reinterpret_cast<const bf16x4_t*>(own_v + 16 * d + 4 * lg);
#pragma unroll
      for (int r = 0; r < 4; ++r) o[d][r] = (float)v[r];
    }
  }
  char* mine = lds + wave * 32 * PITCH;
  const char* tr = mine + (4 * lg + (hc >> 2)) * PITCH + (hc & 3) * 8;
  auto tile = [&](Tile& t, int k0) {
#pragma unroll
    for (int j = 0; j < VL; ++j) {
      const int c = lane + 64 * j;
      *reinterpret_cast<half8_t*>(mine + (c / CH) * PITCH + (c % CH) * 16) = t.v[j];
    }
    float4_t s[2] = {float4_t{0.f, 0.f, 0.f, 0.f}, float4_t{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int b = 0; b < 2; ++b)
        s[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(t.k[b][ks], qf[ks], s[b], 0, 0, 0);
    fetch(t, k0 + 256);
    // s[b][r]: this lane's head, key k0 + 16 b + 4 lg + r
    float tm = -INFINITY;
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        s[b][r] = k0 + 16 * b + 4 * lg + r < k_end ? s[b][r] * scale_log2 : -INFINITY;
        tm = fmaxf(tm, s[b][r]);
      }
    tm = fmaxf(tm, __shfl_xor(tm, 16, MSA_WAVE));
    tm = fmaxf(tm, __shfl_xor(tm, 32, MSA_WAVE));
    const float mn = fmaxf(mx, tm);  // finite: the tile's first key is visible
    if (__ballot(mn > mx)) {
      const float f = __builtin_amdgcn_exp2f(mx - mn);
      l *= f;
#pragma unroll
      for (int d = 0; d < DW; ++d) o[d] = o[d] * f;
      mx = mn;
    }
    bf16x8_t p;
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float v = __builtin_amdgcn_exp2f(s[b][r] - mx);
        l += v;  // this lane group's keys; the groups are summed at the end
        p[4 * b + r] = (bf16_t)v;
      }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // the wave's values lie in LDS
#pragma unroll
    for (int d = 0; d < DW; ++d)
      o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(read_column8(tr + d * 32, tr + d * 32 + 16 * PITCH),
                                                     p, o[d], 0, 0, 0);
    asm volatile("" ::: "memory");  // and are read before the next ones are written
  };
  for (; base + 128 < k_end; base += 256) {
    tile(t0, base);
    tile(t1, base + 128);
  }
  if (base < k_end) tile(t0, base);
  l += __shfl_xor(l, 16, MSA_WAVE);
  l += __shfl_xor(l, 32, MSA_WAVE);
  // merge the waves: o[d][r] is dimension 16 d + 4 lg + r of head hc
  constexpr int OP = VD + 4;
  __syncthreads();
  float* po = reinterpret_cast<float*>(mine) + hc * OP + 4 * lg;
#pragma unroll
  for (int d = 0; d < DW; ++d) *reinterpret_cast<float4_t*>(po + 16 * d) = o[d];
  if (lg == 0) sm[wave][hc] = mx, sl[wave][hc] = l;
  __syncthreads();
  for (int e = tid; e < 16 * (VD / 4); e += 256) {
    const int h = e / (VD / 4), c = (e % (VD / 4)) * 4;
    if (hb * 16 + h >= per) break;  // h grows with e
    float M4 = sm[0][h];
#pragma unroll
    for (int w = 1; w < 4; ++w) M4 = fmaxf(M4, sm[w][h]);
    float4_t sum = {0.f, 0.f, 0.f, 0.f};
    float L4 = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float f = sm[w][h] > -INFINITY ? __builtin_amdgcn_exp2f(sm[w][h] - M4) : 0.f;
      L4 += f * sl[w][h];
      sum += f * *reinterpret_cast<const float4_t*>(lds + w * 32 * PITCH + (h * OP + c) * 4);
    }
    const int hh = g * per + hb * 16 + h;
    if (a.splits > 1) {
      float* p = a.partial + (((int64_t)mr * a.heads + hh) * a.splits + split) * (VD + 4);
      *reinterpret_cast<float4_t*>(p + c) = sum;
      if (c == 0) p[VD] = M4, p[VD + 1] = L4;
    } else {
      const float f = L4 > 0.f ? head_gate(a, m, hh) / L4 : 0.f;
      const int at = hh * VD + c;
      *reinterpret_cast<bf16x4_t*>((bf16_t*)a.out + (a.out_mb > 0
                                                         ? packed_act_offset((int)m, at, a.out_mb)
                                                         : m * a.ldo + at)) =
          bf16x4_t{(bf16_t)(sum[0] * f), (bf16_t)(sum[1] * f), (bf16_t)(sum[2] * f),
                   (bf16_t)(sum[3] * f)};
    }
  }
}

// sums the splits (at most 64) of one (token, head): lane s weighs split s
__global__ __launch_bounds__(64) void grouped_combine_kernel(msa_grouped_args a, int r0) {
  const int64_t row = blockIdx.x;
  const int64_t m = r0 + row / a.heads;
  const int h = (int)(row % a.heads), vd = a.vd, lane = threadIdx.x;
  const float* p = a.partial + row * a.splits * (vd + 4);
  const float* mine = p + (int64_t)min(lane, a.splits - 1) * (vd + 4) + vd;
  const float pm = lane < a.splits ? mine[0] : -INFINITY, pl = mine[1];
  const float gate = head_gate(a, m, h);
  const float mx = wave_max(pm);
  const float w = pm > -INFINITY ? __builtin_amdgcn_exp2f(pm - mx) : 0.f;
  const float l = wave_sum(w * pl);
  const float f = l > 0.f ? gate * w / l : 0.f;  // the split's weight in the output
  for (int c0 = 0; c0 < vd; c0 += 256) {
    const int c = c0 + lane * 4;
    float4_t v = {0.f, 0.f, 0.f, 0.f};
    for (int s0 = 0; s0 < a.splits; s0 += 8) {
      float4_t x[8];
#pragma unroll
      for (int s = 0; s < 8; ++s)
        x[s] = *reinterpret_cast<const float4_t*>(p + (int64_t)min(s0 + s, a.splits - 1) * (vd + 4) +
                                                  min(c, vd - 4));
#pragma unroll
      for (int s = 0; s < 8; ++s) {
        const float ws = __shfl(f, min(s0 + s, 63), MSA_WAVE);
        if (ws != 0.f) v += ws * x[s];  // lanes past the splits weigh nothing
      }
    }
    const int at = h * vd + c;
    if (c < vd)
      *reinterpret_cast<bf16x4_t*>((bf16_t*)a.out + (a.out_mb > 0
                                                         ? packed_act_offset((int)m, at, a.out_mb)
                                                         : m * a.ldo + at)) =
          bf16x4_t{(bf16_t)v[0], (bf16_t)v[1], (bf16_t)v[2], (bf16_t)v[3]};
  }
}

// ---- several new tokens per sequence, bf16 ------------------------------------------------------
constexpr int GF_BM = 128, GF_BN = 64;
template <int HD, int VD>
constexpr int gf_lds_bytes = 2 * GF_BN * (HD * 2 + 16 + VD * 2 + 16);

template <int HD, int VD>
__global__ __launch_bounds__(256) void grouped_flash_kernel(msa_grouped_args a,
                                                            const int32_t* __restrict__ seg_start,
                                                            const int32_t* __restrict__ seg_slot,
                                                            const int32_t* __restrict__ seg_pos,
                                                            int seg0, float scale_log2, int n_qt) {
  constexpr int KSTEPS = HD / 16, DBLK = VD / 32, KP = HD * 2 + 16, VP = VD * 2 + 16;
  constexpr int KT = GF_BN * KP, TILE = KT + GF_BN * VP;
  constexpr int KCH = HD / 8, VCH = VD / 8, KLD = GF_BN * KCH / 256, VLD = GF_BN * VCH / 256;
  extern __shared__ __attribute__((aligned(16))) char lds[];  // [2][K tile, V tile]
  const int seg = seg0 + blockIdx.y, first = seg_start[seg], T = seg_start[seg + 1] - first;
  const int pos0 = seg_pos[seg];
  const int L = blockIdx.x, xcd = L & 7, seq = L >> 3;
  const int hi = seq / n_qt, qt = n_qt - 1 - seq % n_qt;
  if (pos0 < 0 || qt * GF_BM >= T) return;
  // the heads of a group on one XCD where the groups fill the XCDs evenly
  const int per = a.heads / a.kv_heads;
  const int h = a.kv_heads % 8 == 0 ? ((hi / per) * 8 + xcd) * per + hi % per : hi * 8 + xcd;
  if (h >= a.heads) return;
  const int g = h / per;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int j = lane & 31, hl = lane >> 5;
  const int q0 = qt * GF_BM + wave * 32;
  const int tq = q0 + j, tqc = min(tq, T - 1), pq = pos0 + tqc;
  const int lo_q = chunk_start(pq, a.chunk);
  const int k_end = pos0 + min(T, qt * GF_BM + GF_BM);     // behind the last visible key
  const int k_lo = chunk_start(pos0 + qt * GF_BM, a.chunk);  // the first visible key
  const int ntiles = (k_end - k_lo + GF_BN - 1) / GF_BN;
  // what the wave's queries see together, and what each of them sees
  const int w_first = pos0 + min(q0, T - 1), w_last = pos0 + min(q0 + 31, T - 1);
  const int any_lo = chunk_start(w_first, a.chunk), all_lo = chunk_start(w_last, a.chunk);
  const int64_t slot = (int64_t)seg_slot[seg] * a.kv_heads + g;
  const int cs0 = chunk_start(pos0, a.chunk);
  const bf16_t* kc = (const bf16_t*)a.k_cache + slot * a.rows * HD;
  const bf16_t* vc = (const bf16_t*)a.v_cache + slot * a.rows * VD;
  const bf16_t* kn = (const bf16_t*)a.k + (int64_t)first * a.ld + g * HD;
  const bf16_t* vn = (const bf16_t*)a.v + (int64_t)first * a.ld + g * VD;

  bf16x8_t qf[KSTEPS];
  {
    const bf16_t* qr = (const bf16_t*)a.q + (int64_t)(first + tqc) * a.ld + (int64_t)h * HD + hl * 8;
#pragma unroll
    for (int ks = 0; ks < KSTEPS; ++ks) qf[ks] = *reinterpret_cast<const bf16x8_t*>(qr + ks * 16);
  }
  half8_t pk[KLD], pv[VLD];
  auto fetch = [&](int tile) {
#pragma unroll
    for (int i = 0; i < KLD; ++i) {
      const int c = tid + 256 * i, key = min(k_lo + tile * GF_BN + c / KCH, k_end - 1);
      const bf16_t* p = key >= pos0 ? kn + (int64_t)(key - pos0) * a.ld : kc + (int64_t)(key - cs0) * HD;
      pk[i] = *reinterpret_cast<const half8_t*>(p + (c % KCH) * 8);
    }
#pragma unroll
    for (int i = 0; i < VLD; ++i) {
      const int c = tid + 256 * i, key = min(k_lo + tile * GF_BN + c / VCH, k_end - 1);
      const bf16_t* p = key >= pos0 ? vn + (int64_t)(key - pos0) * a.ld : vc + (int64_t)(key - cs0) * VD;
      pv[i] = *reinterpret_cast<const half8_t*>(p + (c % VCH) * 8);
    }
  };
  auto park = [&](int slot) {
    char* kt = lds + slot * TILE;
#pragma unroll
    for (int i = 0; i < KLD; ++i) {
      const int c = tid + 256 * i;
      *reinterpret_cast<half8_t*>(kt + (c / KCH) * KP + (c % KCH) * 16) = pk[i];
    }
#pragma unroll
    for (int i = 0; i < VLD; ++i) {
      const int c = tid + 256 * i;
      *reinterpret_cast<half8_t*>(kt + KT + (c / VCH) * VP + (c % VCH) * 16) = pv[i];
    }
  };
  float16_t o[DBLK];
#pragma unroll
  for (int d = 0; d < DBLK; ++d)
#pragma unroll
    for (int v = 0; v < 16; ++v) o[d][v] = 0.f;
  float mx = -INFINITY, l = 0.f;
  const float16_t zero16 = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f,
                            0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
  // transposing read of V: key row 4 (lane / 32) + (lane % 16) / 4, columns 16 ((lane / 16) % 2) + 4 (lane % 4)
  const int vat = (4 * hl + ((lane & 15) >> 2)) * VP + ((lane >> 4) & 1) * 32 + (lane & 3) * 8;
  fetch(0);
  park(0);
  if (ntiles > 1) fetch(1);
  lds_barrier();
  for (int tile = 0; tile < ntiles; ++tile) {
    const int buf = tile & 1;
    const char* kt = lds + buf * TILE;
    const char* vt = kt + KT;
    if (tile + 1 < ntiles) park(buf ^ 1);
    if (tile + 2 < ntiles) fetch(tile + 2);
    const int kt0 = k_lo + tile * GF_BN;
    // wave-uniform: some query of this wave sees the tile
    if (q0 < T && kt0 <= w_last && kt0 + GF_BN > any_lo) {
      float16_t s[2];
#pragma unroll
      for (int ks = 0; ks < KSTEPS; ++ks)
#pragma unroll
        for (int ib = 0; ib < 2; ++ib) {
          const bf16x8_t x = *reinterpret_cast<const bf16x8_t*>(kt + (ib * 32 + j) * KP + ks * 32 + hl * 16);
          s[ib] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(x, qf[ks], ks == 0 ? zero16 : s[ib], 0, 0, 0);
        }
      // s[ib][v]: key kt0 + 32 ib + 8 (v / 4) + 4 hl + v % 4
      if (kt0 + GF_BN - 1 > w_first || kt0 < all_lo) {
#pragma unroll
        for (int ib = 0; ib < 2; ++ib)
#pragma unroll
          for (int v = 0; v < 16; ++v) {
            const int key = kt0 + ib * 32 + 8 * (v >> 2) + 4 * hl + (v & 3);
            if (key > pq || key < lo_q) s[ib][v] = -INFINITY;
          }
      }
      float tm = s[0][0];
#pragma unroll
      for (int ib = 0; ib < 2; ++ib)
#pragma unroll
        for (int v = 0; v < 16; ++v) tm = fmaxf(tm, s[ib][v]);
      tm = fmaxf(tm, __shfl_xor(tm, 32, MSA_WAVE));
      const float mn = fmaxf(mx, tm * scale_log2);  // scale_log2 > 0
      if (__ballot(mn > mx)) {
        const float f = mx > -INFINITY ? __builtin_amdgcn_exp2f(mx - mn) : 0.f;
        l *= f;
#pragma unroll
        for (int d = 0; d < DBLK; ++d)
#pragma unroll
          for (int v = 0; v < 16; ++v) o[d][v] *= f;
        mx = mn;
      }
      const float base = mx > -INFINITY ? mx : 0.f;
      float t4[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ib = 0; ib < 2; ++ib)
#pragma unroll
        for (int c = 0; c < 2; ++c) {
          bf16x8_t p;
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            const float x = __builtin_amdgcn_exp2f(__builtin_fmaf(s[ib][8 * c + e], scale_log2, -base));
            t4[e & 3] += x;
            p[e] = (bf16_t)x;
          }
#pragma unroll
          for (int d = 0; d < DBLK; ++d) {
            const char* vp = vt + (ib * 32 + c * 16) * VP + vat + d * 64;
            o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(read_column8(vp, vp + 8 * VP), p, o[d], 0, 0,
                                                           0);
          }
        }
      l += (t4[0] + t4[1]) + (t4[2] + t4[3]);
    }
    lds_barrier();
  }
  l += __shfl_xor(l, 32, MSA_WAVE);
  if (tq < T) {
    const int64_t row = first + tq;
    const float inv = l > 0.f ? head_gate(a, row, h) / l : 0.f;
#pragma unroll
    for (int d = 0; d < DBLK; ++d)
#pragma unroll
      for (int blk = 0; blk < 4; ++blk) {
        bf16x4_t v;
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = (bf16_t)(o[d][4 * blk + r] * inv);
        const int c = h * VD + d * 32 + blk * 8 + hl * 4;
        *reinterpret_cast<bf16x4_t*>((bf16_t*)a.out + (a.out_mb > 0
                                                           ? packed_act_offset((int)row, c, a.out_mb)
                                                           : row * a.ldo + c)) = v;
      }
  }
}

// ---- any head size, both formats ----------------------------------------------------------------
constexpr int GS_KEYS = 256;

template <typename T>
__global__ __launch_bounds__(256) void grouped_simple_kernel(msa_grouped_args a, int r0,
                                                             const int32_t* __restrict__ tok_slot,
                                                             const int32_t* __restrict__ tok_pos,
                                                             const int32_t* __restrict__ tok_off) {
  __shared__ float sc[GS_KEYS], red[16], ql[GA_MAX_HEAD];
  const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int64_t m = r0 + blockIdx.y;
  const int pos = tok_pos[m], hd = a.hd, vd = a.vd, g = h / (a.heads / a.kv_heads);
  const int c0 = chunk_start(max(pos, 0), a.chunk), n_keys = pos < 0 ? 0 : pos - c0 + 1;
  const int cached = pos - tok_off[m] - c0;  // keys in front of this step
  const int64_t slot = (int64_t)tok_slot[m] * a.kv_heads + g;
  auto row = [&](const void* cache, const void* rows, int size, int i) {
    return i < cached ? (const T*)cache + (slot * a.rows + i) * size
                      : (const T*)rows + (m - (n_keys - 1 - i)) * a.ld + g * size;
  };
  for (int c = tid; c < hd; c += 256) ql[c] = (float)((const T*)a.q)[m * a.ld + h * hd + c];
  __syncthreads();
  float mx = -INFINITY, l = 0.f, acc[GA_MAX_HEAD / 256];
#pragma unroll
  for (int i = 0; i < GA_MAX_HEAD / 256; ++i) acc[i] = 0.f;
  for (int k0 = 0; k0 < n_keys; k0 += GS_KEYS) {
    const int n = min(GS_KEYS, n_keys - k0);
    for (int k = wave; k < n; k += 4) {
      const T* r = row(a.k_cache, a.k, hd, k0 + k);
      float d = 0.f;
      for (int c = lane; c < hd; c += 64) d = fmaf((float)r[c], ql[c], d);
      d = wave_sum(d);
      if (lane == 0) sc[k] = d * a.scale;
    }
    __syncthreads();
    const float s = tid < n ? sc[tid] : -INFINITY;
    const float mn = fmaxf(mx, block_max(s, red));
    const float e = tid < n ? expf(s - mn) : 0.f;
    const float f = mx > -INFINITY ? expf(mx - mn) : 0.f;
    l = l * f + block_sum(e, red);
    sc[tid] = e;
    mx = mn;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < GA_MAX_HEAD / 256; ++i) {
      const int c = tid + 256 * i;
      if (c >= vd) break;
      float x = acc[i] * f;
      for (int k = 0; k < n; ++k) x = fmaf(sc[k], (float)row(a.v_cache, a.v, vd, k0 + k)[c], x);
      acc[i] = x;
    }
    __syncthreads();
  }
  const float f = l > 0.f ? head_gate(a, m, h) / l : 0.f;
#pragma unroll
  for (int i = 0; i < GA_MAX_HEAD / 256; ++i) {
    const int c = tid + 256 * i;
    if (c >= vd) break;
    const int at = h * vd + c;
    ((T*)a.out)[a.out_mb > 0 ? packed_act_offset((int)m, at, a.out_mb) : m * a.ldo + at] =
        (T)(acc[i] * f);
  }
}

bool tile_size(int n) { return n == 64 || n == 128 || n == 192 || n == 256; }
bool has_tiles(const msa_grouped_args& a) {
  return a.dtype == MSA_BF16 && tile_size(a.hd) && tile_size(a.vd);
}

template <int HD, int VD, bool FUSED>
bool run_decode(const msa_grouped_args& a, const msa_batch* b, int r0, int segs, hipStream_t s) {
  static std::atomic<uint64_t> raised{0};
  constexpr int bytes = gd_lds_bytes<HD, VD>;
  if (!raise_lds((const void*)grouped_decode_kernel<HD, VD, FUSED>, bytes, raised)) return false;
  const int HB = (a.heads / a.kv_heads + 15) / 16;
  hipLaunchKernelGGL((grouped_decode_kernel<HD, VD, FUSED>),
                     dim3((unsigned)(segs * a.kv_heads * HB * a.splits)), dim3(256), bytes, s, a, r0, segs,
                     b->tok_slot, b->tok_pos, a.scale * LOG2E);
  return true;
}

template <int HD, int VD>
bool run_tiles(const msa_grouped_args& a, const msa_batch* b, int r0, int seg0, int segs, int longest,
               hipStream_t s) {
  if (longest == 1) {
    const bool ok = a.fused ? run_decode<HD, VD, true>(a, b, r0, segs, s)
                            : run_decode<HD, VD, false>(a, b, r0, segs, s);
    if (!ok) return false;
    if (a.splits > 1)
      hipLaunchKernelGGL(grouped_combine_kernel, dim3((unsigned)(segs * a.heads)), dim3(64), 0, s, a, r0);
    return true;
  }
  static std::atomic<uint64_t> raised{0};
  constexpr int bytes = gf_lds_bytes<HD, VD>;
  if (!raise_lds((const void*)grouped_flash_kernel<HD, VD>, bytes, raised)) return false;
  const int n_qt = (longest + GF_BM - 1) / GF_BM;
  hipLaunchKernelGGL((grouped_flash_kernel<HD, VD>), dim3((unsigned)((a.heads + 7) / 8 * 8 * n_qt), segs),
                     dim3(256), bytes, s, a, b->seg_start, b->seg_slot, b->seg_pos, seg0,
                     a.scale * LOG2E, n_qt);
  return true;
}

template <int HD>
bool run_head(const msa_grouped_args& a, const msa_batch* b, int r0, int seg0, int segs, int longest,
              hipStream_t s) {
  switch (a.vd) {
    case 64: return run_tiles<HD, 64>(a, b, r0, seg0, segs, longest, s);
    case 128: return run_tiles<HD, 128>(a, b, r0, seg0, segs, longest, s);
    case 192: return run_tiles<HD, 192>(a, b, r0, seg0, segs, longest, s);
    case 256: return run_tiles<HD, 256>(a, b, r0, seg0, segs, longest, s);
  }
  return false;
}

int check_grouped(const char* name, const msa_grouped_args* a, const msa_batch* b) {
  MSA_REQUIRE(a && b && a->q && a->k && a->v && a->k_cache && a->v_cache &&
                  (a->rot_dims == 0 || a->inv_freq),
              MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  MSA_REQUIRE(a->heads > 0 && a->kv_heads > 0 && a->heads % a->kv_heads == 0 && a->hd > 0 &&
                  a->hd % 16 == 0 && a->hd <= GA_MAX_HEAD && a->vd > 0 && a->vd % 16 == 0 &&
                  a->vd <= GA_MAX_HEAD && a->chunk >= 0 && a->rot_dims >= 0 && a->rot_dims % 2 == 0 &&
                  a->rot_dims <= a->hd && a->rows > 0 && a->ld % 8 == 0,
              MSA_ERR_INVALID_ARG, "%s: heads=%d kv_heads=%d sizes %d and %d (at most %d) rot_dims=%d rows=%d",
              name, a->heads, a->kv_heads, a->hd, a->vd, GA_MAX_HEAD, a->rot_dims, a->rows);
  MSA_REQUIRE(b->M > 0 && b->M <= 65535 && b->nseg > 0 && b->nseg <= 65535, MSA_ERR_INVALID_ARG,
              "%s: %d tokens in %d segments", name, b->M, b->nseg);
  return MSA_OK;
}

}  // namespace

extern "C" int msa_grouped_rotate(const msa_grouped_args* a, const msa_batch* b, void* stream) {
  const char* name = "msa_grouped_rotate";
  int rc = check_grouped(name, a, b);
  if (rc) return rc;
  const int append = b->max_count == 1, half = a->rot_dims / 2;
  if (!append && half == 0) return MSA_OK;
#define GR_RUN(T, V)                                                                              \
  hipLaunchKernelGGL((rotate_kernel<T, V>), dim3(b->M), dim3(256), 0, (hipStream_t)stream, *a,    \
                     b->tok_slot, b->tok_pos, append)
  if (a->dtype == MSA_BF16) {
    if (half % 8 == 0) GR_RUN(bf16_t, 8);
    else GR_RUN(bf16_t, 1);
  } else {
    if (half % 4 == 0) GR_RUN(float, 4);
    else GR_RUN(float, 1);
  }
#undef GR_RUN
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_grouped_append(const msa_grouped_args* a, const msa_batch* b, void* stream) {
  const char* name = "msa_grouped_append";
  int rc = check_grouped(name, a, b);
  if (rc) return rc;
  if (b->max_count == 1) return MSA_OK;
  const int most = a->chunk > 0 && a->chunk < b->max_count ? a->chunk : b->max_count;
  const dim3 grid((most + AP_TOK - 1) / AP_TOK, b->nseg);
  if (a->dtype == MSA_BF16)
    hipLaunchKernelGGL(append_kernel<bf16_t>, grid, dim3(256), 0, (hipStream_t)stream, *a, b->seg_start,
                       b->seg_slot, b->seg_pos);
  else
    hipLaunchKernelGGL(append_kernel<float>, grid, dim3(256), 0, (hipStream_t)stream, *a, b->seg_start,
                       b->seg_slot, b->seg_pos);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_grouped_attention_splits(const msa_grouped_args* a, int M, int key_bound) {
  if (!a || M < 1 || key_bound < 1 || !has_tiles(*a)) return 1;
  const int per = a->heads / a->kv_heads;
  const int64_t groups = (int64_t)M * a->kv_heads * ((per + 15) / 16);
  const int keys = a->chunk > 0 && a->chunk < key_bound ? a->chunk : key_bound;
  int s = 1;
  // up to a workgroup per CU, at least 128 keys (a tile per wave) each
  while (s < 64 && groups * s * 2 <= 256 && (int64_t)keys >= 256 * s) s *= 2;
  return s;
}

extern "C" int msa_grouped_fuses(const msa_grouped_args* a, const msa_batch* b) {
  return a && b && b->max_count == 1 && has_tiles(*a);
}

extern "C" int msa_grouped_attention(const msa_grouped_args* a, const msa_batch* b, int seg0, int seg1,
                                     int longest, void* stream) {
  const char* name = "msa_grouped_attention";
  int rc = check_grouped(name, a, b);
  if (rc) return rc;
  MSA_REQUIRE(seg0 >= 0 && seg0 < seg1 && seg1 <= b->nseg && longest >= 1 && longest <= b->max_count,
              MSA_ERR_INVALID_ARG, "%s: segments %d .. %d of %d, up to %d tokens", name, seg0, seg1,
              b->nseg, longest);
  MSA_REQUIRE(a->out && a->scale > 0.f && a->splits >= 1 && a->splits <= 64 &&
                  (a->splits == 1 || (a->partial && longest == 1 && has_tiles(*a))),
              MSA_ERR_INVALID_ARG, "%s: splits=%d scale=%g", name, a->splits, (double)a->scale);
  MSA_REQUIRE(b->max_count == 1 || b->host_start, MSA_ERR_INVALID_ARG, "%s: no host tables", name);
  MSA_REQUIRE(!a->fused || msa_grouped_fuses(a, b), MSA_ERR_INVALID_ARG, "%s: nothing to fuse with", name);
  hipStream_t s = (hipStream_t)stream;
  const int r0 = b->max_count == 1 ? seg0 : b->host_start[seg0];
  const int r1 = b->max_count == 1 ? seg1 : b->host_start[seg1];
  if (has_tiles(*a)) {
    bool ok = false;
    switch (a->hd) {
      case 64: ok = run_head<64>(*a, b, r0, seg0, seg1 - seg0, longest, s); break;
      case 128: ok = run_head<128>(*a, b, r0, seg0, seg1 - seg0, longest, s); break;
      case 192: ok = run_head<192>(*a, b, r0, seg0, seg1 - seg0, longest, s); break;
      case 256: ok = run_head<256>(*a, b, r0, seg0, seg1 - seg0, longest, s); break;
    }
    MSA_REQUIRE(ok, MSA_ERR_HIP, "%s: LDS limit", name);
  } else {
    const dim3 grid(a->heads, r1 - r0);
    if (a->dtype == MSA_BF16)
      hipLaunchKernelGGL(grouped_simple_kernel<bf16_t>, grid, dim3(256), 0, s, *a, r0, b->tok_slot,
                         b->tok_pos, b->tok_off);
    else
      hipLaunchKernelGGL(grouped_simple_kernel<float>, grid, dim3(256), 0, s, *a, r0, b->tok_slot,
                         b->tok_pos, b->tok_off);
  }
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}
