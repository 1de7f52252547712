// Causal softmax attention over a cached latent (keys and values are both linear images of one
// vector per position, which is all that is cached).
//
//  * Few new tokens per sequence (decode): the query is multiplied by the key up-projection
//    first, so that scores are dot products with the latent itself, and the value up-projection is
//    applied to the weighted sum of latents.  All heads share the latent rows: a workgroup takes
//    64 positions at a time into LDS once and uses them twice, row-wise for the scores and through
//    the transposing LDS read for the weighted sum.  Bound: the latent rows from HBM, once per 32
//    heads; the workgroups of one token's head groups and key range run on one XCD.
//  * Prompts: keys and values are expanded per head and flash_attention_kernel runs over them.
#include <math.h>

#include "attention_tiles.h"

namespace {

constexpr int LA_KEYS = 64, LA_SC = LA_KEYS + 4;  // keys per tile; pitch of a head's scores
template <int RP>
constexpr int la_tile_bytes = LA_KEYS * (RP * 2 + 16);
template <int RP, int NHB>
constexpr int la_lds_bytes = la_tile_bytes<RP> + NHB * 16 * LA_SC * 4;

// ---- few new tokens, bf16 --------------------------------------------------------------------
// A workgroup owns one token, one range of keys and NHB blocks of 16 heads, four waves per block.
// The four waves share the scores of a 64-key tile (16 keys each) through LDS and then the weighted
// sum by latent dimensions (RP / 4 each), so that no wave holds more than its share of the
// accumulators and nothing has to be merged at the end.  The rows of the next two tiles are on their way
// into registers while a tile is worked on.
template <int RP, int NHB>
__global__ __launch_bounds__(256 * NHB) void latent_decode_kernel(
    const bf16_t* __restrict__ q, const bf16_t* __restrict__ latent, int capacity, int heads,
    float scale_log2, bf16_t* __restrict__ out, float* __restrict__ partial, int splits,
    const int32_t* __restrict__ tok_slot, const int32_t* __restrict__ tok_pos, int M) {
  constexpr int KS = RP / 32, DW = RP / 64, PITCH = RP * 2 + 16, THREADS = 256 * NHB;
  constexpr int CH = RP / 8, LD = LA_KEYS * CH / THREADS;  // 16-byte chunks of a row; loads per thread
  extern __shared__ __attribute__((aligned(16))) char lds[];  // tile, then scores [NHB][16][LA_SC]
  const int HG = (heads + 16 * NHB - 1) / (16 * NHB);
  // workgroup -> (token, split, head group): the head groups of one (token, split) on one XCD
  const int L = blockIdx.x, xcd = L & 7, seq = L >> 3;
  const int pair = (seq / HG) * 8 + xcd, hg = seq % HG;
  if (pair >= M * splits) return;
  const int m = pair / splits, split = pair - m * splits;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int w4 = wave & 3, hb = wave >> 2;
  const int hc = lane & 15, g = lane >> 4;  // head column, lane group
  const int head = (hg * NHB + hb) * 16 + hc;
  const int n_keys = min(tok_pos[m] + 1, capacity);  // <= 0: inactive
  const int per = split_keys(n_keys, splits);
  const int k_begin = split * per, k_end = min(n_keys, k_begin + per);
  const bf16_t* rows = latent + (int64_t)tok_slot[m] * capacity * RP;

  half8_t pre0[LD], pre1[LD];
  auto fetch = [&](half8_t(&pre)[LD], int k0) {
#pragma unroll
    for (int i = 0; i < LD; ++i) {
      const int c = tid + THREADS * i;
      const int key = min(k0 + c / CH, n_keys - 1);
      pre[i] = *reinterpret_cast<const half8_t*>(rows + (int64_t)key * RP + (c % CH) * 8);
    }
  };
  bf16x8_t qf[KS];
  {
    const bf16_t* qr = q + ((int64_t)m * heads + min(head, heads - 1)) * RP + g * 8;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) qf[ks] = *reinterpret_cast<const bf16x8_t*>(qr + ks * 32);
  }
  if (k_begin < k_end) {
    fetch(pre0, k_begin);
    fetch(pre1, k_begin + LA_KEYS);  // past the end: the last key again
  }
  // the queries have arrived here: a wait for them inside the loop would, on every pass, also be
  // one for the tiles in flight
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) asm volatile("" : "+v"(qf[ks]));
  float4_t o[DW];
#pragma unroll
  for (int d = 0; d < DW; ++d) o[d] = float4_t{0.f, 0.f, 0.f, 0.f};
  float mx = -INFINITY, l = 0.f;
  float* sc = reinterpret_cast<float*>(lds + la_tile_bytes<RP>) + (hb * 16 + hc) * LA_SC;
  const char* krow = lds + (16 * w4 + hc) * PITCH + g * 16;
  // transposing reads: lane (g, i) is the source of key row 4 g + i / 4, columns 4 (i % 4) ..
  const char* tr = lds + (4 * g + (hc >> 2)) * PITCH + w4 * (RP / 2) + (hc & 3) * 8;
  auto tile = [&](half8_t(&pre)[LD], int k0) {
    lds_barrier();  // the previous tile and its scores are consumed
#pragma unroll
    for (int i = 0; i < LD; ++i) {
      const int c = tid + THREADS * i;
      *reinterpret_cast<half8_t*>(lds + (c / CH) * PITCH + (c % CH) * 16) = pre[i];
    }
    // (past the end: the last key again - an unconditional load keeps the count of loads in flight
    // known, so that the wait for one tile's rows is not a wait for the next one's)
    fetch(pre, k0 + 2 * LA_KEYS);
    lds_barrier();
    float4_t s2[2] = {float4_t{0.f, 0.f, 0.f, 0.f}, float4_t{0.f, 0.f, 0.f, 0.f}};
    constexpr int PD = 4;  // key fragments read ahead
    bf16x8_t ka[PD];
#pragma unroll
    for (int ks = 0; ks < PD; ++ks) ka[ks] = *reinterpret_cast<const bf16x8_t*>(krow + ks * 64);
    __builtin_amdgcn_sched_group_barrier(0x100, PD, 0);
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const bf16x8_t cur = ka[ks % PD];
      s2[ks & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cur, qf[ks], s2[ks & 1], 0, 0, 0);
      __builtin_amdgcn_sched_group_barrier(0x008, 1, 0);
      if (ks + PD < KS) {
        ka[ks % PD] = *reinterpret_cast<const bf16x8_t*>(krow + (ks + PD) * 64);
        __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
      }
    }
    float4_t s = s2[0] + s2[1];
    // s[r]: this lane's head, key k0 + 16 w4 + 4 g + r
#pragma unroll
    for (int r = 0; r < 4; ++r)
      s[r] = k0 + 16 * w4 + 4 * g + r < k_end ? s[r] * scale_log2 : -INFINITY;
    *reinterpret_cast<float4_t*>(sc + 16 * w4 + 4 * g) = s;
    lds_barrier();
    // every wave of a head block: the lane's keys 32 t + 4 g + {0 .. 3}, 32 t + 16 + 4 g + {0 .. 3}
    float4_t e[2][2];
    float tm = -INFINITY;
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        e[t][b] = *reinterpret_cast<const float4_t*>(sc + 32 * t + 16 * b + 4 * g);
        tm = fmaxf(fmaxf(tm, fmaxf(e[t][b][0], e[t][b][1])), fmaxf(e[t][b][2], e[t][b][3]));
      }
    tm = fmaxf(tm, __shfl_xor(tm, 16, MSA_WAVE));
    tm = fmaxf(tm, __shfl_xor(tm, 32, MSA_WAVE));
    const float mn = fmaxf(mx, tm);  // finite: the first tile's first key is visible
    if (__ballot(mn > mx)) {
      const float f = __builtin_amdgcn_exp2f(mx - mn);
      l *= f;
#pragma unroll
      for (int d = 0; d < DW; ++d) o[d] = o[d] * f;
      mx = mn;
    }
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      bf16x8_t p;
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float v = __builtin_amdgcn_exp2f(e[t][b][r] - mx);
          l += v;  // this lane group's keys; the groups are summed at the end
          p[4 * b + r] = (bf16_t)v;
        }
#pragma unroll
      for (int d = 0; d < DW; ++d) {
        const char* a = tr + 32 * t * PITCH + d * 32;
        o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(read_column8(a, a + 16 * PITCH), p, o[d], 0,
                                                       0, 0);
      }
    }
  };
  int k0 = k_begin;
  for (; k0 + LA_KEYS < k_end; k0 += 2 * LA_KEYS) {
    tile(pre0, k0);
    tile(pre1, k0 + LA_KEYS);
  }
  if (k0 < k_end) tile(pre0, k0);
  l += __shfl_xor(l, 16, MSA_WAVE);
  l += __shfl_xor(l, 32, MSA_WAVE);
  if (head >= heads) return;
  // o[d][r]: dimension w4 RP / 4 + 16 d + 4 g + r
  const int64_t row = (int64_t)m * heads + head;
  const int c0 = w4 * (RP / 4) + 4 * g;
  if (splits > 1) {
    float* p = partial + (row * splits + split) * (RP + 4);
#pragma unroll
    for (int d = 0; d < DW; ++d) *reinterpret_cast<float4_t*>(p + c0 + 16 * d) = o[d];
    if (w4 == 0 && g == 0) p[RP] = mx, p[RP + 1] = l;
  } else {
    const float inv = l > 0.f ? 1.f / l : 0.f;
#pragma unroll
    for (int d = 0; d < DW; ++d)
      *reinterpret_cast<bf16x4_t*>(out + row * RP + c0 + 16 * d) =
          bf16x4_t{(bf16_t)(o[d][0] * inv), (bf16_t)(o[d][1] * inv), (bf16_t)(o[d][2] * inv),
                   (bf16_t)(o[d][3] * inv)};
  }
}

// ---- any rank, both formats: one workgroup per (token, head, split), vector ALU ---------------
constexpr int LS_KEYS = 256, LS_MAX_RP = 2048;

template <typename T>
__global__ __launch_bounds__(256) void latent_simple_kernel(
    const T* __restrict__ q, const T* __restrict__ latent, int capacity, int heads, int rp,
    float scale, T* __restrict__ out, float* __restrict__ partial, int splits,
    const int32_t* __restrict__ tok_slot, const int32_t* __restrict__ tok_pos) {
  __shared__ float sc[LS_KEYS], red[16], ql[LS_MAX_RP];
  const int h = blockIdx.x, m = blockIdx.y, split = blockIdx.z, tid = threadIdx.x, lane = tid & 63,
            wave = tid >> 6;
  const int n_keys = min(tok_pos[m] + 1, capacity);
  const int per = split_keys(n_keys, splits);
  const int k_begin = split * per, k_end = min(n_keys, k_begin + per);
  const T* rows = latent + (int64_t)tok_slot[m] * capacity * rp;
  const int64_t row = (int64_t)m * heads + h;
  for (int c = tid; c < rp; c += 256) ql[c] = (float)q[row * rp + c];
  __syncthreads();
  float mx = -INFINITY, l = 0.f, acc[LS_MAX_RP / 256];
#pragma unroll
  for (int i = 0; i < LS_MAX_RP / 256; ++i) acc[i] = 0.f;
  for (int k0 = k_begin; k0 < k_end; k0 += LS_KEYS) {
    const int n = min(LS_KEYS, k_end - k0);
    for (int k = wave; k < n; k += 4) {
      const T* r = rows + (int64_t)(k0 + k) * rp;
      float d = 0.f;
      for (int c = lane; c < rp; c += 64) d = fmaf((float)r[c], ql[c], d);
      d = wave_sum(d);
      if (lane == 0) sc[k] = d * scale;
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
    for (int i = 0; i < LS_MAX_RP / 256; ++i) {
      const int c = tid + 256 * i;
      if (c >= rp) break;
      float a = acc[i] * f;
      for (int k = 0; k < n; ++k) a = fmaf(sc[k], (float)rows[(int64_t)(k0 + k) * rp + c], a);
      acc[i] = a;
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < LS_MAX_RP / 256; ++i) {
    const int c = tid + 256 * i;
    if (c >= rp) break;
    if (splits > 1)
      partial[(row * splits + split) * (rp + 4) + c] = acc[i];
    else
      out[row * rp + c] = (T)(l > 0.f ? acc[i] / l : 0.f);
  }
  if (splits > 1 && tid == 0) {
    float* p = partial + (row * splits + split) * (rp + 4) + rp;
    p[0] = mx * LOG2E, p[1] = l;  // maxima travel in units of log 2
  }
}

// sums the splits of one (token, head)
template <typename T>
__global__ __launch_bounds__(128) void latent_combine_kernel(const float* __restrict__ partial,
                                                             int splits, int rp, T* __restrict__ out) {
  const int64_t row = blockIdx.x;
  const float* p = partial + row * splits * (rp + 4);
  float mx = -INFINITY;
  for (int s = 0; s < splits; ++s) mx = fmaxf(mx, p[(int64_t)s * (rp + 4) + rp]);
  float l = 0.f;
  for (int s = 0; s < splits; ++s) {
    const float* q = p + (int64_t)s * (rp + 4) + rp;
    if (q[0] > -INFINITY) l += __builtin_amdgcn_exp2f(q[0] - mx) * q[1];
  }
  const float inv = l > 0.f ? 1.f / l : 0.f;
  for (int c = threadIdx.x * 4; c < rp; c += 512) {
    float4_t a = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < splits; ++s) {
      const float* q = p + (int64_t)s * (rp + 4);
      if (q[rp] > -INFINITY)
        a += __builtin_amdgcn_exp2f(q[rp] - mx) * *reinterpret_cast<const float4_t*>(q + c);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) out[row * rp + c + i] = (T)(a[i] * inv);
  }
}

// ---- prompts: flash attention over expanded keys and values ------------------------------------
// 128 queries of one head per workgroup, 4 waves x 32 queries, key tiles of 64, one pass with an
// online softmax.  Everything is transposed (S^T = K Q^T, O^T = V^T P^T) so that a query's scores lie
// in one lane (and its partner 32 lanes away) and P^T is the B operand as it stands.  Tiles go
// through registers into LDS rows padded by 16 bytes, one tile ahead, double buffered.  The query
// tiles of one head run on one XCD, the longest first.
constexpr int FA_BM = 128, FA_BN = 64;
template <int HD>
constexpr int fa_pitch = HD * 2 + 16;
template <int HD>
constexpr int fa_lds_bytes = 2 * 2 * FA_BN * fa_pitch<HD>;

template <int HD>
__global__ __launch_bounds__(256) void flash_attention_kernel(
    const bf16_t* __restrict__ q, int64_t ldq, const bf16_t* __restrict__ kv, int64_t ldkv,
    bf16_t* __restrict__ out, int64_t ldo, int out_mb, int row0, int heads, int T, int pos0,
    float scale_log2, int n_qt) {
  constexpr int KSTEPS = HD / 16, DBLK = HD / 32, PITCH = fa_pitch<HD>, TILE = FA_BN * PITCH;
  constexpr int CH = HD / 8, LD = FA_BN * CH / 256;  // chunks per row; loads per thread and tile
  extern __shared__ __attribute__((aligned(16))) char lds[];  // [2][K, V][TILE]
  const int L = blockIdx.x, xcd = L & 7, seq = L >> 3;
  const int h = (seq / n_qt) * 8 + xcd, qt = n_qt - 1 - seq % n_qt;
  if (h >= heads) return;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int j = lane & 31, hl = lane >> 5;
  const int q0 = qt * FA_BM + wave * 32;
  const int tq = q0 + j, tqc = min(tq, T - 1), pq = pos0 + tqc;
  const int n_keys = pos0 + min(T, qt * FA_BM + FA_BM);
  const int ntiles = (n_keys + FA_BN - 1) / FA_BN;
  const bf16_t* kb = kv + (int64_t)h * HD;
  const bf16_t* vb = kv + (int64_t)(heads + h) * HD;

  bf16x8_t qf[KSTEPS];
  {
    const bf16_t* qr = q + (int64_t)tqc * ldq + (int64_t)h * HD + hl * 8;
#pragma unroll
    for (int ks = 0; ks < KSTEPS; ++ks) qf[ks] = *reinterpret_cast<const bf16x8_t*>(qr + ks * 16);
  }
  half8_t pk[LD], pv[LD];
  auto fetch = [&](int tile) {
#pragma unroll
    for (int i = 0; i < LD; ++i) {
      const int c = tid + 256 * i;
      const int64_t key = min(tile * FA_BN + c / CH, n_keys - 1);
      pk[i] = *reinterpret_cast<const half8_t*>(kb + key * ldkv + (c % CH) * 8);
      pv[i] = *reinterpret_cast<const half8_t*>(vb + key * ldkv + (c % CH) * 8);
    }
  };
  auto park = [&](int slot) {
    char* kt = lds + slot * 2 * TILE;
#pragma unroll
    for (int i = 0; i < LD; ++i) {
      const int c = tid + 256 * i, at = (c / CH) * PITCH + (c % CH) * 16;
      *reinterpret_cast<half8_t*>(kt + at) = pk[i];
      *reinterpret_cast<half8_t*>(kt + TILE + at) = pv[i];
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
  const int vat = (4 * hl + ((lane & 15) >> 2)) * PITCH + ((lane >> 4) & 1) * 32 + (lane & 3) * 8;
  fetch(0);
  park(0);
  if (ntiles > 1) fetch(1);
  lds_barrier();
  for (int tile = 0; tile < ntiles; ++tile) {
    const int slot = tile & 1;
    const char* kt = lds + slot * 2 * TILE;
    const char* vt = kt + TILE;
    if (tile + 1 < ntiles) park(slot ^ 1);
    if (tile + 2 < ntiles) fetch(tile + 2);
    const int kt0 = tile * FA_BN;
    if (kt0 <= pos0 + q0 + 31) {  // wave-uniform: some query of this wave sees the tile
      float16_t s[2];
#pragma unroll
      for (int ks = 0; ks < KSTEPS; ++ks)
#pragma unroll
        for (int ib = 0; ib < 2; ++ib) {
          const bf16x8_t a = *reinterpret_cast<const bf16x8_t*>(kt + (ib * 32 + j) * PITCH + ks * 32 +
                                                                hl * 16);
          s[ib] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, qf[ks], ks == 0 ? zero16 : s[ib], 0, 0, 0);
        }
      // s[ib][v]: key kt0 + 32 ib + 8 (v / 4) + 4 hl + v % 4
      if (kt0 + FA_BN - 1 > pos0 + q0) {
#pragma unroll
        for (int ib = 0; ib < 2; ++ib)
#pragma unroll
          for (int v = 0; v < 16; ++v)
            if (kt0 + ib * 32 + 8 * (v >> 2) + 4 * hl + (v & 3) > pq) s[ib][v] = -INFINITY;
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
            const char* vp = vt + (ib * 32 + c * 16) * PITCH + vat + d * 64;
            o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(read_column8(vp, vp + 8 * PITCH), p, o[d],
                                                           0, 0, 0);
          }
        }
      l += (t4[0] + t4[1]) + (t4[2] + t4[3]);
    }
    lds_barrier();
  }
  l += __shfl_xor(l, 32, MSA_WAVE);
  if (tq < T) {
    const float inv = l > 0.f ? 1.f / l : 0.f;
    const int row = row0 + tq;
#pragma unroll
    for (int d = 0; d < DBLK; ++d)
#pragma unroll
      for (int blk = 0; blk < 4; ++blk) {
        bf16x4_t v;
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = (bf16_t)(o[d][4 * blk + r] * inv);
        const int c = h * HD + d * 32 + blk * 8 + hl * 4;
        *reinterpret_cast<bf16x4_t*>(out + (out_mb > 0 ? packed_act_offset(row, c, out_mb)
                                                       : (int64_t)row * ldo + c)) = v;
      }
  }
}

template <int RP, int NHB>
bool run_decode_blocks(const void* q, const void* latent, int capacity, int heads, float scale,
                       void* out, float* partial, int splits, const int32_t* tok_slot,
                       const int32_t* tok_pos, int M, hipStream_t s) {
  static std::atomic<uint64_t> raised{0};
  constexpr int bytes = la_lds_bytes<RP, NHB>;
  if (!raise_lds((const void*)latent_decode_kernel<RP, NHB>, bytes, raised)) return false;
  const int HG = (heads + 16 * NHB - 1) / (16 * NHB);
  const int64_t groups = ((int64_t)M * splits + 7) / 8 * 8 * HG;
  hipLaunchKernelGGL((latent_decode_kernel<RP, NHB>), dim3((unsigned)groups), dim3(256 * NHB), bytes,
                     s, (const bf16_t*)q, (const bf16_t*)latent, capacity, heads, scale * LOG2E,
                     (bf16_t*)out, partial, splits, tok_slot, tok_pos, M);
  return true;
}

template <int RP>
bool run_decode(const void* q, const void* latent, int capacity, int heads, float scale, void* out,
                float* partial, int splits, const int32_t* tok_slot, const int32_t* tok_pos, int M,
                hipStream_t s) {
  return heads <= 16 ? run_decode_blocks<RP, 1>(q, latent, capacity, heads, scale, out, partial,
                                                splits, tok_slot, tok_pos, M, s)
                     : run_decode_blocks<RP, 2>(q, latent, capacity, heads, scale, out, partial,
                                                splits, tok_slot, tok_pos, M, s);
}

bool has_decode_kernel(int dtype, int rp) {
  return dtype == MSA_BF16 && (rp == 128 || rp == 192 || rp == 256 || rp == 384 || rp == 512);
}

template <int HD>
bool run_flash(const void* q, int64_t ldq, const void* kv, int64_t ldkv, void* out, int64_t ldo,
               int out_mb, int row0, int heads, int T, int pos0, float scale, hipStream_t s) {
  static std::atomic<uint64_t> raised{0};
  if (!raise_lds((const void*)flash_attention_kernel<HD>, fa_lds_bytes<HD>, raised)) return false;
  const int n_qt = (T + FA_BM - 1) / FA_BM;
  hipLaunchKernelGGL(flash_attention_kernel<HD>, dim3((unsigned)((heads + 7) / 8 * 8 * n_qt)),
                     dim3(256), fa_lds_bytes<HD>, s, (const bf16_t*)q, ldq, (const bf16_t*)kv, ldkv,
                     (bf16_t*)out, ldo, out_mb, row0, heads, T, pos0, scale * LOG2E, n_qt);
  return true;
}

}  // namespace

extern "C" int msa_latent_attention_splits(int dtype, int M, int heads, int rp, int key_bound) {
  if (M < 1 || heads < 1 || key_bound < 1) return 1;
  const int64_t groups = (int64_t)M * (has_decode_kernel(dtype, rp) ? (heads + 31) / 32 : heads);
  int s = 1;
  // about a workgroup per CU, at least 128 keys each
  while (s < 64 && groups * s < 256 && (int64_t)key_bound >= 256 * s) s *= 2;
  return s;
}

extern "C" int msa_latent_attention(int dtype, const void* q, const void* latent, int capacity,
                                    int heads, int rp, float scale, void* out, float* partial,
                                    int splits, const int32_t* tok_slot, const int32_t* tok_pos,
                                    int M, void* stream) {
  const char* name = "msa_latent_attention";
  MSA_REQUIRE(q && latent && out && tok_slot && tok_pos && (splits == 1 || partial),
              MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  MSA_REQUIRE(M > 0 && M <= 65535 && heads > 0 && rp > 0 && rp % 8 == 0 && rp <= LS_MAX_RP &&
                  capacity > 0 && splits >= 1 && splits <= 64,
              MSA_ERR_INVALID_ARG, "%s: M=%d heads=%d rp=%d (at most %d) splits=%d", name, M, heads, rp,
              LS_MAX_RP, splits);
  MSA_REQUIRE(scale > 0.f, MSA_ERR_INVALID_ARG, "%s: scale must be positive", name);
  hipStream_t s = (hipStream_t)stream;
  if (has_decode_kernel(dtype, rp)) {
    bool ok = false;
#define LA_CASE(RP)                                                                                 \
  case RP:                                                                                          \
    ok = run_decode<RP>(q, latent, capacity, heads, scale, out, partial, splits, tok_slot, tok_pos, \
                        M, s);                                                                      \
    break;
    switch (rp) {
      LA_CASE(128)
      LA_CASE(192)
      LA_CASE(256)
      LA_CASE(384)
      LA_CASE(512)
    }
#undef LA_CASE
    MSA_REQUIRE(ok, MSA_ERR_HIP, "%s: LDS limit", name);
  } else {
    const dim3 grid(heads, M, splits);
    if (dtype == MSA_BF16)
      hipLaunchKernelGGL(latent_simple_kernel<bf16_t>, grid, dim3(256), 0, s, (const bf16_t*)q,
                         (const bf16_t*)latent, capacity, heads, rp, scale, (bf16_t*)out, partial,
                         splits, tok_slot, tok_pos);
    else
      hipLaunchKernelGGL(latent_simple_kernel<float>, grid, dim3(256), 0, s, (const float*)q,
                         (const float*)latent, capacity, heads, rp, scale, (float*)out, partial,
                         splits, tok_slot, tok_pos);
  }
  if (splits > 1) {
    if (dtype == MSA_BF16)
      hipLaunchKernelGGL(latent_combine_kernel<bf16_t>, dim3((unsigned)(M * heads)), dim3(128), 0, s,
                         partial, splits, rp, (bf16_t*)out);
    else
      hipLaunchKernelGGL(latent_combine_kernel<float>, dim3((unsigned)(M * heads)), dim3(128), 0, s,
                         partial, splits, rp, (float*)out);
  }
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_flash_attention_bf16(const void* q, int64_t ldq, const void* kv, int64_t ldkv,
                                        void* out, int64_t ldo, int out_mb, int row0, int heads, int hd,
                                        int T, int pos0, float scale, void* stream) {
  const char* name = "msa_flash_attention_bf16";
  MSA_REQUIRE(q && kv && out, MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  MSA_REQUIRE(T > 0 && pos0 >= 0 && row0 >= 0 && heads > 0 && ldq % 8 == 0 && ldkv % 8 == 0 &&
                  ldkv >= 2 * (int64_t)heads * hd && ldq >= (int64_t)heads * hd && scale > 0.f &&
                  (out_mb == 0 || row0 + T <= out_mb * 16),
              MSA_ERR_INVALID_ARG, "%s: T=%d pos0=%d heads=%d hd=%d", name, T, pos0, heads, hd);
  bool ok = false;
#define FA_CASE(HD)                                                                                \
  case HD:                                                                                         \
    ok = run_flash<HD>(q, ldq, kv, ldkv, out, ldo, out_mb, row0, heads, T, pos0, scale,            \
                       (hipStream_t)stream);                                                       \
    break;
  switch (hd) {
    FA_CASE(32)
    FA_CASE(64)
    FA_CASE(96)
    FA_CASE(128)
    FA_CASE(192)
    FA_CASE(256)
    default:
      msa_set_error("%s: head size %d", name, hd);
      return MSA_ERR_INVALID_ARG;
  }
#undef FA_CASE
  MSA_REQUIRE(ok, MSA_ERR_HIP, "%s: LDS limit", name);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}
