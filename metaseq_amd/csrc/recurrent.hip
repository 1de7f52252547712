// Recurrent mixers over flat batches of segments: the short causal convolution, the gated linear
// recurrent unit and the gated delta rule.  All state is fp32 and lives per cache slot; a segment
// whose first position is 0 starts from zero whatever the slot held before.
#include <math.h>

#include "common.h"

namespace {

template <typename T>
struct Vec8 {
  typedef T type __attribute__((ext_vector_type(8), aligned(16)));
};

__device__ __forceinline__ float silu(float v) { return v / (1.f + expf(-v)); }
__device__ __forceinline__ float gate_of(float v, int act) {
  return (act == MSA_GATE_SIGMOID ? 1.f : v) / (1.f + expf(-v));
}
// ---- short convolution ----------------------------------------------------------------------
constexpr int SC_TOK = 8;      // tokens per workgroup
constexpr int SC_MAX_TAPS = 8;

// A thread owns 8 channels of SC_TOK tokens.  STEP: one token per segment; the thread also shifts
// the state.  TAPS > 0: that many taps, and a tile that lies inside one segment behind its first
// TAPS - 1 tokens (nearly every tile of a prompt) requests all its input rows at once; the other tiles
// take every input from the segment or the state, tap by tap.
template <typename T, bool STEP, int TAPS>
__global__ __launch_bounds__(256) void short_conv_kernel(
    const T* __restrict__ in, int64_t ld_in, int C, int taps, const float* __restrict__ in_bias,
    const float* __restrict__ weight, const float* __restrict__ bias, int act, T* __restrict__ out,
    int64_t ld_out, T* __restrict__ state, const int32_t* __restrict__ tok_slot,
    const int32_t* __restrict__ tok_pos, const int32_t* __restrict__ tok_off, int M) {
  typedef typename Vec8<T>::type v8;
  const int c = (blockIdx.x * 256 + threadIdx.x) * 8;
  if (c >= C) return;
  const int m0 = blockIdx.y * (STEP ? 1 : SC_TOK), m1 = min(M, m0 + (STEP ? 1 : SC_TOK));
  float ib[8], b[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    ib[i] = in_bias ? in_bias[c + i] : 0.f;
    b[i] = bias ? bias[c + i] : 0.f;
  }
  if constexpr (!STEP && TAPS > 1) {
    const int off = tok_off[m0];
    if (m1 - m0 == SC_TOK && off >= TAPS - 1 && tok_pos[m0] >= 0 &&
        tok_off[m1 - 1] - off == SC_TOK - 1) {
      v8 x[SC_TOK + TAPS - 1];
#pragma unroll
      for (int t = 0; t < SC_TOK + TAPS - 1; ++t)
        x[t] = *reinterpret_cast<const v8*>(in + (int64_t)(m0 - (TAPS - 1) + t) * ld_in + c);
      float w[TAPS][8];
#pragma unroll
      for (int j = 0; j < TAPS; ++j)
#pragma unroll
        for (int i = 0; i < 8; ++i) w[j][i] = weight[(int64_t)j * C + c + i];
#pragma unroll
      for (int t = 0; t < SC_TOK; ++t) {
        v8 o;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          float a = b[i];
#pragma unroll
          for (int j = 0; j < TAPS; ++j) a = fmaf((float)x[t + j][i] + ib[i], w[j][i], a);
          o[i] = (T)(act ? silu(a) : a);
        }
        *reinterpret_cast<v8*>(out + (int64_t)(m0 + t) * ld_out + c) = o;
      }
      return;
    }
  }
  for (int m = m0; m < m1; ++m) {
    const int pos = tok_pos[m], off = tok_off[m];
    T* st = state + ((int64_t)tok_slot[m] * (taps - 1)) * C + c;
    float a[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) a[i] = b[i];
    for (int lag = taps - 1; lag >= 0; --lag) {
      if (pos - lag < 0) continue;  // before the start (or an inactive token)
      const v8 v = lag <= off ? *reinterpret_cast<const v8*>(in + (int64_t)(m - lag) * ld_in + c)
                              : *reinterpret_cast<const v8*>(st + (int64_t)(taps - 1 - (lag - off)) * C);
      const float* w = weight + (int64_t)(taps - 1 - lag) * C + c;
#pragma unroll
      for (int i = 0; i < 8; ++i) a[i] = fmaf((float)v[i] + ib[i], w[i], a[i]);
      if (STEP && lag < taps - 1)  // the state row in front of the one this lag came from
        *reinterpret_cast<v8*>(st + (int64_t)(taps - 2 - lag) * C) = v;
    }
    v8 o;
#pragma unroll
    for (int i = 0; i < 8; ++i) o[i] = (T)(act ? silu(a[i]) : a[i]);
    *reinterpret_cast<v8*>(out + (int64_t)m * ld_out + c) = o;
  }
}

// state after the segment: row j holds the input of position end - (taps - 1) + j
template <typename T>
__global__ __launch_bounds__(256) void conv_state_kernel(
    const T* __restrict__ in, int64_t ld_in, int C, int taps, T* __restrict__ state,
    const int32_t* __restrict__ seg_start, const int32_t* __restrict__ seg_slot,
    const int32_t* __restrict__ seg_pos) {
  const int c = blockIdx.x * 256 + threadIdx.x, s = blockIdx.y;
  if (c >= C || seg_pos[s] < 0) return;
  const int first = seg_start[s], n = seg_start[s + 1] - first;
  T* st = state + (int64_t)seg_slot[s] * (taps - 1) * C + c;
  // rows move towards the front only, so they can be written in increasing order
  for (int j = 0; j < taps - 1; ++j) {
    const int t = n - (taps - 1) + j;  // offset in the segment; negative: in the old state
    st[(int64_t)j * C] = t >= 0 ? in[(int64_t)(first + t) * ld_in + c]
                                : st[(int64_t)(t + taps - 1) * C];
  }
}

// ---- gated linear recurrent unit ------------------------------------------------------------
constexpr int RG_CHUNK = 32;

// log a and the input term of one (token, channel)
__device__ __forceinline__ void rglru_terms(float gr, float gi, float rate, float u, float& a, float& b) {
  const float log_a = -8.f * sigmoidf(gr) * rate;
  a = expf(log_a);
  b = sqrtf(-expm1f(2.f * log_a)) * sigmoidf(gi) * u;
}

// pass 1: a and b of every token in place of the gates, and the chunk's (product of a, end state
// from zero)
template <typename T>
__global__ __launch_bounds__(256) void rglru_local_kernel(
    float* __restrict__ gates, const float* __restrict__ gate_bias, const float* __restrict__ lam,
    const T* __restrict__ u, int64_t ld_u, int C, float* __restrict__ carry, int chunks,
    const int32_t* __restrict__ seg_start) {
  const int c = blockIdx.x * 256 + threadIdx.x, ch = blockIdx.y, s = blockIdx.z;
  if (c >= C) return;
  const int first = seg_start[s] + ch * RG_CHUNK, end = min(seg_start[s + 1], first + RG_CHUNK);
  if (first >= end) return;
  const float rate = softplus(lam[c]), br = gate_bias[c], bi = gate_bias[C + c];
  float A = 1.f, S = 0.f;
  for (int m = first; m < end; ++m) {
    float* g = gates + (int64_t)m * 2 * C + c;
    float a, b;
    rglru_terms(g[0] + br, g[C] + bi, rate, (float)u[(int64_t)m * ld_u + c], a, b);
    g[0] = a, g[C] = b;
    A *= a;
    S = fmaf(a, S, b);
  }
  float* k = carry + (((int64_t)s * chunks + ch) * 2) * C + c;
  k[0] = A, k[C] = S;
}

// pass 2: the state in front of the chunk from the slot's state and the carries of the chunks
// before it, then the outputs.  DIRECT: no pass 1, one chunk covers the segment.
template <typename T, bool DIRECT>
__global__ __launch_bounds__(256) void rglru_output_kernel(
    const float* __restrict__ gates, const float* __restrict__ gate_bias,
    const float* __restrict__ lam, const T* __restrict__ u, int64_t ld_u, const T* __restrict__ y,
    int64_t ld_y, const float* __restrict__ y_bias, int C, float* __restrict__ state,
    const float* __restrict__ carry, int chunks, T* __restrict__ out, int64_t ld_out, int out_mb,
    const int32_t* __restrict__ seg_start, const int32_t* __restrict__ seg_slot,
    const int32_t* __restrict__ seg_pos) {
  const int c = blockIdx.x * 256 + threadIdx.x, ch = blockIdx.y, s = blockIdx.z;
  if (c >= C) return;
  const int n = seg_start[s + 1] - seg_start[s];
  const int first = seg_start[s] + (DIRECT ? 0 : ch * RG_CHUNK);
  const int end = DIRECT ? seg_start[s + 1] : min(seg_start[s + 1], first + RG_CHUNK);
  if (first >= end) return;
  const int pos = seg_pos[s];
  float* slot = state + (int64_t)seg_slot[s] * C + c;
  float S = pos > 0 ? *slot : 0.f;
  if (!DIRECT) {
    const float* k = carry + (int64_t)s * chunks * 2 * C + c;
    for (int j = 0; j < ch; ++j) S = fmaf(k[(int64_t)j * 2 * C], S, k[(int64_t)j * 2 * C + C]);
  }
  float rate = 0.f, br = 0.f, bi = 0.f;
  if (DIRECT) rate = softplus(lam[c]), br = gate_bias[c], bi = gate_bias[C + c];
  const float yb = y_bias[c];
  for (int m = first; m < end; ++m) {
    const float* g = gates + (int64_t)m * 2 * C + c;
    float a = g[0], b = g[C];
    if (DIRECT) rglru_terms(g[0] + br, g[C] + bi, rate, (float)u[(int64_t)m * ld_u + c], a, b);
    S = fmaf(a, S, b);
    const float o = S * gelu_tanh((float)y[(int64_t)m * ld_y + c] + yb);
    out[out_mb > 0 ? packed_act_offset(m, c, out_mb) : (int64_t)m * ld_out + c] = (T)o;
  }
  // the state is read by every chunk of the segment in this launch: only with one chunk may the
  // same launch write it (rglru_state_kernel otherwise)
  if ((DIRECT || n <= RG_CHUNK) && pos >= 0) *slot = S;
}

__global__ __launch_bounds__(256) void rglru_state_kernel(
    int C, float* __restrict__ state, const float* __restrict__ carry, int chunks,
    const int32_t* __restrict__ seg_start, const int32_t* __restrict__ seg_slot,
    const int32_t* __restrict__ seg_pos) {
  const int c = blockIdx.x * 256 + threadIdx.x, s = blockIdx.y;
  if (c >= C || seg_pos[s] < 0) return;
  const int n = seg_start[s + 1] - seg_start[s], used = (n + RG_CHUNK - 1) / RG_CHUNK;
  if (used <= 1) return;
  float* slot = state + (int64_t)seg_slot[s] * C + c;
  float S = seg_pos[s] > 0 ? *slot : 0.f;
  const float* k = carry + (int64_t)s * chunks * 2 * C + c;
  for (int j = 0; j < used; ++j) S = fmaf(k[(int64_t)j * 2 * C], S, k[(int64_t)j * 2 * C + C]);
  *slot = S;
}

// ---- gated delta rule -------------------------------------------------------------------------
// Every column of a head's state evolves by itself (given k and q), so a workgroup owns one
// segment, one head and 256 / LPC of its columns: LPC lanes hold a column, each R consecutive rows of
// it in registers, through all tokens of the segment.  16 lanes per column spread a single
// prompt over the chip; 8 need fewer instructions per column where there are segments enough.  With S the state before the
// token's decay, one pass over it yields both products the token needs:
//   u = beta (v - g S^T k),   o = S_new^T q = g S^T q + u (k . q),   S_new = g S + k u^T.
// CH: one decay per key channel (a row of S), taken from `decay`; S is decayed before the pass.
// Tokens are taken DR_TOK at a time: the next chunk's rows are fetched into registers while the
// current chunk runs out of LDS, where k and q arrive as unit vectors.
constexpr int DR_TOK = 16;

__device__ __forceinline__ float row16_sum(float v) {
  v += dpp_move<0xB1, 0xf>(0.f, v);
  v += dpp_move<0x4E, 0xf>(0.f, v);
  v += dpp_move<0x124, 0xf>(0.f, v);
  v += dpp_move<0x128, 0xf>(0.f, v);
  return v;
}

template <int LPC>
__device__ __forceinline__ float lanes_sum(float v) {  // over LPC = 8 or 16 neighbouring lanes
  if constexpr (LPC == 16) return row16_sum(v);
  v += dpp_move<0xB1, 0xf>(0.f, v);
  v += dpp_move<0x4E, 0xf>(0.f, v);
  v += dpp_move<0x141, 0xf>(0.f, v);  // row_half_mirror: the other quad of the eight
  return v;
}

template <typename T, int DP, int LPC, bool CH>
__global__ __launch_bounds__(256) void delta_scan_kernel(
    const T* __restrict__ qkv, int64_t ld, const float* __restrict__ ba, int ldba,
    const float* __restrict__ decay_rate, const float* __restrict__ dt_bias,
    const float* __restrict__ decay, int heads, int kv_heads, float q_scale, int vp, float* __restrict__ state, float* __restrict__ o,
    const int32_t* __restrict__ seg_start, const int32_t* __restrict__ seg_slot,
    const int32_t* __restrict__ seg_pos) {
  constexpr int R = DP / LPC, CW = 256 / LPC, R16 = DP / 16;
  __shared__ __attribute__((aligned(16))) float lk[DR_TOK][DP], lq[DR_TOK][DP],
      ld_[CH ? DR_TOK : 1][CH ? DP : 4];
  __shared__ float lv[DR_TOK][CW], lo[DR_TOK][CW], lg[DR_TOK], lb[DR_TOK], lkq[DR_TOK];
  const int s = blockIdx.z, h = blockIdx.y, col0 = blockIdx.x * CW;
  const int tid = threadIdx.x;
  const int first = seg_start[s], n = seg_start[s + 1] - first, pos = seg_pos[s];
  const int hk = h / (heads / kv_heads);
  const int q_at = hk * DP, k_at = kv_heads * DP + hk * DP, v_at = 2 * kv_heads * DP + h * vp + col0;
  if (pos < 0) {
    for (int i = tid; i < n * CW; i += 256)
      o[(int64_t)(first + i / CW) * heads * vp + h * vp + col0 + i % CW] = 0.f;
    return;
  }
  const int cl = tid / LPC, rl = tid % LPC;  // column of the workgroup's, row group
  float* st = state + (((int64_t)seg_slot[s] * heads + h) * vp + col0 + cl) * DP + rl * R;
  float S[R];
#pragma unroll
  for (int i = 0; i < R; ++i) S[i] = pos > 0 ? st[i] : 0.f;
  const float rate = CH ? 0.f : decay_rate[h], dtb = CH ? 0.f : dt_bias[h];

  // staging: vector x = tid / 8 (tokens 0 .. 15 of q, then of k), elements EV * (tid % 8) ..
  constexpr int EV = DP / 8, VPT = DR_TOK * CW / 256;  // q or k elements, v elements per thread
  constexpr int GV = CH ? (DR_TOK * DP + 1023) / 1024 : 0;  // decays per thread, four at a time
  const int sv = tid >> 3, stok = sv & 15, sel = (tid & 7) * EV;
  const bool is_k = sv >= 16;
  T raw[EV];
  float rv[VPT], rb = 0.f, rg = 0.f;
  float4_t rd[GV > 0 ? GV : 1];
  auto fetch = [&](int t0) {
    const int t = min(t0 + stok, n - 1);
    const T* p = qkv + (int64_t)(first + t) * ld + (is_k ? k_at : q_at) + sel;
    typedef T t4 __attribute__((ext_vector_type(4), aligned(8)));
#pragma unroll
    for (int i = 0; i < EV; i += 4) {
      const t4 x = *reinterpret_cast<const t4*>(p + i);
#pragma unroll
      for (int j = 0; j < 4; ++j) raw[i + j] = x[j];
    }
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int e = tid + 256 * i, tv = min(t0 + e / CW, n - 1);
      rv[i] = (float)qkv[(int64_t)(first + tv) * ld + v_at + e % CW];
    }
    if (tid < DR_TOK) {
      const float* z = ba + (int64_t)(first + min(t0 + tid, n - 1)) * ldba;
      rb = z[h];
      if (!CH) rg = z[heads + h];
    }
#pragma unroll
    for (int i = 0; i < GV; ++i) {
      const int e = min((tid + 256 * i) * 4, DR_TOK * DP - 4), t = min(t0 + e / DP, n - 1);
      rd[i] = *reinterpret_cast<const float4_t*>(decay + ((int64_t)(first + t) * heads + h) * DP +
                                                 e % DP);
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < n; t0 += DR_TOK) {
    const int nt = min(DR_TOK, n - t0);
    {
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < EV; ++i) ss += (float)raw[i] * (float)raw[i];
      ss += __shfl_xor(ss, 1, MSA_WAVE);
      ss += __shfl_xor(ss, 2, MSA_WAVE);
      ss += __shfl_xor(ss, 4, MSA_WAVE);
      const float f = (is_k ? 1.f : q_scale) / sqrtf(ss + 1e-6f);
      float* dst = (is_k ? lk[stok] : lq[stok]) + sel;
#pragma unroll
      for (int i = 0; i < EV; ++i) dst[i] = (float)raw[i] * f;
#pragma unroll
      for (int i = 0; i < VPT; ++i) (&lv[0][0])[tid + 256 * i] = rv[i];
      if (tid < DR_TOK) {
        lb[tid] = sigmoidf(rb);
        if (!CH) lg[tid] = decay_of(rg + dtb, rate);
      }
#pragma unroll
      for (int i = 0; i < GV; ++i)
        if ((tid + 256 * i) * 4 < DR_TOK * DP)
          *reinterpret_cast<float4_t*>(&ld_[0][0] + (tid + 256 * i) * 4) = rd[i];
    }
    lds_barrier();
    {
      const int t = tid >> 4, r = tid & 15;
      float d = 0.f;
#pragma unroll
      for (int i = 0; i < R16; ++i) d = fmaf(lk[t][r * R16 + i], lq[t][r * R16 + i], d);
      d = row16_sum(d);
      if (r == 0) lkq[t] = d;
    }
    if (t0 + DR_TOK < n) fetch(t0 + DR_TOK);  // in flight across the barriers
    lds_barrier();
    // operands of the current and the next token: one set is fetched while the other is used
    struct Token {
      float k[R], q[R], d[CH ? R : 1], g, beta, v, kq;
    } a, b;
    auto read = [&](Token& x, int t) {
      t = min(t, DR_TOK - 1);
#pragma unroll
      for (int i = 0; i < R; ++i) x.k[i] = lk[t][rl * R + i], x.q[i] = lq[t][rl * R + i];
      if constexpr (CH) {
#pragma unroll
        for (int i = 0; i < R; ++i) x.d[i] = ld_[t][rl * R + i];
      }
      x.g = CH ? 1.f : lg[t], x.beta = lb[t], x.v = lv[t][cl], x.kq = lkq[t];
    };
    auto advance = [&](const Token& x, int t) {
      float d1 = 0.f, d2 = 0.f, e1 = 0.f, e2 = 0.f;
      if constexpr (CH) {
#pragma unroll
        for (int i = 0; i < R; ++i) S[i] *= x.d[i];
      }
#pragma unroll
      for (int i = 0; i < R; i += 2) {
        d1 = fmaf(S[i], x.k[i], d1);
        e1 = fmaf(S[i + 1], x.k[i + 1], e1);
        d2 = fmaf(S[i], x.q[i], d2);
        e2 = fmaf(S[i + 1], x.q[i + 1], e2);
      }
      d1 = lanes_sum<LPC>(d1 + e1);
      d2 = lanes_sum<LPC>(d2 + e2);
      const float u = x.beta * (x.v - (CH ? d1 : x.g * d1));
#pragma unroll
      for (int i = 0; i < R; ++i) S[i] = fmaf(x.k[i], u, CH ? S[i] : x.g * S[i]);
      if (rl == 0) lo[t][cl] = fmaf(u, x.kq, CH ? d2 : x.g * d2);
    };
    read(a, 0);
    for (int t = 0; t < nt; t += 2) {
      read(b, t + 1);
      advance(a, t);
      read(a, t + 2);
      if (t + 1 < nt) advance(b, t + 1);
    }
    lds_barrier();
    for (int e = tid; e < nt * CW; e += 256)
      o[(int64_t)(first + t0 + e / CW) * heads * vp + h * vp + col0 + e % CW] = (&lo[0][0])[e];
  }
#pragma unroll
  for (int i = 0; i < R; ++i) st[i] = S[i];
}

// One token per segment (a decode step): a workgroup owns one segment and one head with all its
// columns, 4 CG of them per wave and pass, requests the whole pass's state at once and finishes the
// head's output (norm over the columns, gate) itself.  Lanes and arithmetic as above.
template <typename T, int R, int CG, bool CH>
__global__ __launch_bounds__(256) void delta_step_kernel(
    const T* __restrict__ qkv, int64_t ld, const float* __restrict__ ba, int ldba,
    const float* __restrict__ decay_rate, const float* __restrict__ dt_bias,
    const float* __restrict__ decay, int heads, int kv_heads, float q_scale, int vdim, int vp,
    float* __restrict__ state, const T* __restrict__ gate, int64_t ld_gate, int gate_act, const float* __restrict__ w, float eps, T* __restrict__ out, int64_t ld_out,
    int out_mb, const int32_t* __restrict__ seg_slot, const int32_t* __restrict__ seg_pos) {
  constexpr int DP = 16 * R;
  __shared__ __attribute__((aligned(16))) float lk[DP], lq[DP];
  __shared__ float lv[512], lo[512], red[16];
  const int m = blockIdx.y, h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int pos = seg_pos[m];
  const int rl = lane & 15, cw = wave * 4 + (lane >> 4);  // row group; column within a group of 16
  float* st = state + (((int64_t)seg_slot[m] * heads + h) * vp) * DP + rl * R;
  const int ng = vp / 16;
  typedef float fr __attribute__((ext_vector_type(2), aligned(8)));
  float S[CG][R];
  auto load = [&](int g0) {
#pragma unroll
    for (int c = 0; c < CG; ++c) {
      const fr* p = reinterpret_cast<const fr*>(st + (int64_t)(min(g0 + c, ng - 1) * 16 + cw) * DP);
#pragma unroll
      for (int i = 0; i < R / 2; ++i) {
        const fr v = p[i];
        S[c][2 * i] = v[0], S[c][2 * i + 1] = v[1];
      }
    }
  };
  load(0);
  const T* row = qkv + (int64_t)m * ld;
  const int hk = h / (heads / kv_heads);
  if (wave < 2) {  // q and k as unit vectors
    const T* p = row + (wave == 0 ? hk : kv_heads + hk) * DP;
    float x[(DP + 63) / 64], ss = 0.f;
#pragma unroll
    for (int i = 0; i < (DP + 63) / 64; ++i) {
      const int c = lane + 64 * i;
      x[i] = c < DP ? (float)p[min(c, DP - 1)] : 0.f;
      ss += x[i] * x[i];
    }
    ss = wave_sum(ss);
    const float f = (wave == 0 ? q_scale : 1.f) / sqrtf(ss + 1e-6f);
#pragma unroll
    for (int i = 0; i < (DP + 63) / 64; ++i)
      if (lane + 64 * i < DP) (wave == 0 ? lq : lk)[lane + 64 * i] = x[i] * f;
  } else {
    for (int c = tid - 128; c < vp; c += 128)
      lv[c] = (float)row[2 * kv_heads * DP + h * vp + c];
  }
  const float* z = ba + (int64_t)m * ldba;
  const float bt = sigmoidf(z[h]);
  const float g = CH ? 1.f : decay_of(z[heads + h] + dt_bias[h], decay_rate[h]);
  float gr[CH ? R : 1];  // decays of the lane's rows
  if constexpr (CH) {
    const float* p = decay + ((int64_t)m * heads + h) * DP + rl * R;
#pragma unroll
    for (int i = 0; i < R; ++i) gr[i] = p[i];
  }
  lds_barrier();
  float k[R], q[R], kq = 0.f;
#pragma unroll
  for (int i = 0; i < R; ++i) {
    k[i] = lk[rl * R + i], q[i] = lq[rl * R + i];
    kq = fmaf(k[i], q[i], kq);
  }
  kq = row16_sum(kq);
  for (int g0 = 0; g0 < ng; g0 += CG) {
    if (g0 > 0) load(g0);
#pragma unroll
    for (int c = 0; c < CG; ++c) {
      if (g0 + c >= ng) break;  // uniform
      const int col = (g0 + c) * 16 + cw;
      if (pos <= 0) {
#pragma unroll
        for (int i = 0; i < R; ++i) S[c][i] = 0.f;
      }
      float d1 = 0.f, d2 = 0.f;
      if constexpr (CH) {
#pragma unroll
        for (int i = 0; i < R; ++i) S[c][i] *= gr[i];
      }
#pragma unroll
      for (int i = 0; i < R; ++i) {
        d1 = fmaf(S[c][i], k[i], d1);
        d2 = fmaf(S[c][i], q[i], d2);
      }
      d1 = row16_sum(d1);
      d2 = row16_sum(d2);
      const float u = bt * (lv[col] - g * d1);
      if (rl == 0) lo[col] = fmaf(u, kq, g * d2);
      if (pos >= 0) {
        fr* p = reinterpret_cast<fr*>(st + (int64_t)col * DP);
#pragma unroll
        for (int i = 0; i < R / 2; ++i)
          p[i] = fr{fmaf(k[2 * i], u, g * S[c][2 * i]), fmaf(k[2 * i + 1], u, g * S[c][2 * i + 1])};
      }
    }
  }
  lds_barrier();
  float ss = 0.f;
  for (int c = tid; c < vp; c += 256) ss += lo[c] * lo[c];
  ss = block_sum(ss, red);
  const float rms = 1.f / sqrtf(ss / (float)vdim + eps);
  for (int c = tid; c < vp; c += 256) {
    const int at = h * vp + c;
    const float y = lo[c] * rms * w[c] * gate_of((float)gate[(int64_t)m * ld_gate + at], gate_act);
    out[out_mb > 0 ? packed_act_offset(m, at, out_mb) : (int64_t)m * ld_out + at] = (T)y;
  }
}

// one wave per (token, head)
template <typename T>
__global__ __launch_bounds__(256) void delta_output_kernel(
    const float* __restrict__ o, const T* __restrict__ gate, int64_t ld_gate, int gate_act,
    const float* __restrict__ w, int heads, int vdim, int vp, float eps, T* __restrict__ out,
    int64_t ld_out, int out_mb, int M) {
  const int64_t idx = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (idx >= (int64_t)M * heads) return;
  const int lane = threadIdx.x & 63;
  const int m = (int)(idx / heads), h = (int)(idx % heads);
  const float* row = o + idx * vp;
  float v[8], ss = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int c = lane + 64 * i;
    v[i] = c < vp ? row[c] : 0.f;
    ss += v[i] * v[i];
  }
  ss = wave_sum(ss);
  const float r = 1.f / sqrtf(ss / (float)vdim + eps);
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int c = lane + 64 * i;
    if (c < vp) {
      const int at = h * vp + c;
      const float y = v[i] * r * w[c] * gate_of((float)gate[(int64_t)m * ld_gate + at], gate_act);
      out[out_mb > 0 ? packed_act_offset(m, at, out_mb) : (int64_t)m * ld_out + at] = (T)y;
    }
  }
}

template <typename T, int DP, int LPC>
void run_delta(const msa_delta_args& a, const msa_batch* b, hipStream_t s) {
  const dim3 grid(a.vp / (256 / LPC), a.heads, b->nseg);
  const float q_scale = (float)pow((double)a.dim, -0.5);
#define DR_RUN(CH)                                                                                 \
  hipLaunchKernelGGL((delta_scan_kernel<T, DP, LPC, CH>), grid, dim3(256), 0, s, (const T*)a.qkv,  \
                     a.ld, a.ba, a.ldba, a.decay_rate, a.dt_bias, a.decay, a.heads, a.kv_heads,    \
                     q_scale, a.vp, a.state, a.o, b->seg_start, b->seg_slot, b->seg_pos)
  if (a.decay) DR_RUN(true);
  else DR_RUN(false);
#undef DR_RUN
}

template <typename T, int DP>
void pick_delta(const msa_delta_args& a, const msa_batch* b, hipStream_t s) {
  // eight lanes per column from two waves per SIMD on (of 1024)
  if (a.vp % 32 == 0 && (int64_t)b->nseg * a.heads * (a.vp / 32) * 4 >= 2048)
    run_delta<T, DP, 8>(a, b, s);
  else
    run_delta<T, DP, 16>(a, b, s);
}

template <typename T, int R, int CG>
void run_delta_step(const msa_delta_args& a, const msa_batch* b, hipStream_t s) {
  const dim3 grid(a.heads, b->nseg);
  const float q_scale = (float)pow((double)a.dim, -0.5);
#define DR_RUN(CH)                                                                                 \
  hipLaunchKernelGGL((delta_step_kernel<T, R, CG, CH>), grid, dim3(256), 0, s, (const T*)a.qkv,    \
                     a.ld, a.ba, a.ldba, a.decay_rate, a.dt_bias, a.decay, a.heads, a.kv_heads,    \
                     q_scale, a.vdim, a.vp, a.state, (const T*)a.gate, a.ld_gate, a.gate_act, a.w, \
                     a.eps, (T*)a.out, a.ld_out, a.out_mb, b->seg_slot, b->seg_pos)
  if (a.decay) DR_RUN(true);
  else DR_RUN(false);
#undef DR_RUN
}

template <typename T>
void dispatch_delta(const msa_delta_args& a, const msa_batch* b, bool step, hipStream_t s) {
#define DR_CASE(DP, CG)                              \
  case DP:                                           \
    if (step) run_delta_step<T, DP / 16, CG>(a, b, s); \
    else pick_delta<T, DP>(a, b, s);                 \
    break;
  switch (a.dp) {
    DR_CASE(32, 8)
    DR_CASE(64, 8)
    DR_CASE(96, 8)
    DR_CASE(128, 8)
    DR_CASE(192, 4)
    DR_CASE(256, 4)
  }
#undef DR_CASE
}

int check_delta(const char* name, const msa_delta_args* a, const msa_batch* b) {
  MSA_REQUIRE(a && b && a->qkv && a->ba && a->state && (a->decay || (a->decay_rate && a->dt_bias)),
              MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  const int dp = a->dp;
  MSA_REQUIRE((dp == 32 || dp == 64 || dp == 96 || dp == 128 || dp == 192 || dp == 256) &&
                  a->dim > 0 && a->dim <= dp && a->vp > 0 && a->vp % 16 == 0 && a->heads > 0 &&
                  a->kv_heads > 0 && a->heads % a->kv_heads == 0 &&
                  a->ldba >= (a->decay ? 1 : 2) * a->heads && a->ld % 8 == 0 && a->heads <= 65535 &&
                  b->nseg > 0 && b->nseg <= 65535,
              MSA_ERR_INVALID_ARG, "%s: heads=%d kv_heads=%d dim=%d dp=%d vp=%d", name, a->heads,
              a->kv_heads, a->dim, dp, a->vp);
  return MSA_OK;
}

}  // namespace

extern "C" int msa_delta_step(const msa_delta_args* a, const msa_batch* b, void* stream) {
  const char* name = "msa_delta_step";
  int rc = check_delta(name, a, b);
  if (rc) return rc;
  MSA_REQUIRE(a->gate && a->w && a->out, MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  MSA_REQUIRE(a->vdim <= a->vp && a->vp <= 512 && b->max_count == 1 && b->M == b->nseg,
              MSA_ERR_INVALID_ARG, "%s: vdim=%d vp=%d, %d tokens in %d segments", name, a->vdim, a->vp,
              b->M, b->nseg);
  if (a->dtype == MSA_BF16)
    dispatch_delta<bf16_t>(*a, b, true, (hipStream_t)stream);
  else
    dispatch_delta<float>(*a, b, true, (hipStream_t)stream);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_short_conv(int dtype, const void* in, int64_t ld_in, int C, int taps,
                              const float* in_bias, const float* weight, const float* bias, int silu,
                              void* out, int64_t ld_out, void* state, const msa_batch* b,
                              void* stream) {
  const char* name = "msa_short_conv";
  MSA_REQUIRE(in && weight && out && b && (state || taps == 1), MSA_ERR_INVALID_ARG,
              "%s: null pointer", name);
  MSA_REQUIRE(C > 0 && C % 8 == 0 && ld_in % 8 == 0 && ld_out % 8 == 0 && taps >= 1 &&
                  taps <= SC_MAX_TAPS && b->M > 0 && b->M <= 65535 * SC_TOK,
              MSA_ERR_INVALID_ARG, "%s: C=%d taps=%d (at most %d) M=%d", name, C, taps, SC_MAX_TAPS,
              b->M);
  const bool step = b->max_count == 1 && b->M <= 65535;
  const dim3 grid((C / 8 + 255) / 256, step ? b->M : (b->M + SC_TOK - 1) / SC_TOK);
#define SC_RUN(T, STEP, TAPS)                                                                       \
  hipLaunchKernelGGL((short_conv_kernel<T, STEP, TAPS>), grid, dim3(256), 0, (hipStream_t)stream,   \
                     (const T*)in, ld_in, C, taps, in_bias, weight, bias, silu, (T*)out, ld_out,    \
                     (T*)state, b->tok_slot, b->tok_pos, b->tok_off, b->M)
#define SC_TYPE(T)                                                                                  \
  do {                                                                                              \
    if (step) SC_RUN(T, true, 0);                                                                   \
    else if (taps == 2) SC_RUN(T, false, 2);                                                        \
    else if (taps == 3) SC_RUN(T, false, 3);                                                        \
    else if (taps == 4) SC_RUN(T, false, 4);                                                        \
    else SC_RUN(T, false, 0);                                                                       \
  } while (0)
  if (dtype == MSA_BF16) SC_TYPE(bf16_t);
  else SC_TYPE(float);
#undef SC_TYPE
#undef SC_RUN
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_conv_state(int dtype, const void* in, int64_t ld_in, int C, int taps, void* state,
                              const msa_batch* b, void* stream) {
  const char* name = "msa_conv_state";
  MSA_REQUIRE(in && b && (state || taps == 1), MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  if (taps == 1 || (b->max_count == 1 && b->M <= 65535)) return MSA_OK;  // nothing, or done
  MSA_REQUIRE(b->nseg <= 65535, MSA_ERR_INVALID_ARG, "%s: too many segments", name);
  const dim3 grid((C + 255) / 256, b->nseg);
  if (dtype == MSA_BF16)
    hipLaunchKernelGGL(conv_state_kernel<bf16_t>, grid, dim3(256), 0, (hipStream_t)stream,
                       (const bf16_t*)in, ld_in, C, taps, (bf16_t*)state, b->seg_start, b->seg_slot,
                       b->seg_pos);
  else
    hipLaunchKernelGGL(conv_state_kernel<float>, grid, dim3(256), 0, (hipStream_t)stream,
                       (const float*)in, ld_in, C, taps, (float*)state, b->seg_start, b->seg_slot,
                       b->seg_pos);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_rglru_chunks(int max_count) { return (max_count + RG_CHUNK - 1) / RG_CHUNK; }

extern "C" int msa_rglru_scan(int dtype, float* gates, const float* gate_bias, const float* lam,
                              const void* u, int64_t ld_u, const void* y, int64_t ld_y,
                              const float* y_bias, int C, float* state, float* carry, void* out,
                              int64_t ld_out, int out_mb, const msa_batch* b, void* stream) {
  const char* name = "msa_rglru_scan";
  MSA_REQUIRE(gates && gate_bias && lam && u && y && y_bias && state && out && b, MSA_ERR_INVALID_ARG,
              "%s: null pointer", name);
  const int chunks = msa_rglru_chunks(b->max_count);
  MSA_REQUIRE(C > 0 && b->nseg > 0 && b->nseg <= 65535 && chunks >= 1 && chunks <= 65535 &&
                  (chunks == 1 || carry),
              MSA_ERR_INVALID_ARG, "%s: C=%d nseg=%d chunks=%d", name, C, b->nseg, chunks);
  hipStream_t s = (hipStream_t)stream;
  const dim3 grid((C + 255) / 256, chunks, b->nseg);
#define RG_RUN(T)                                                                                   \
  if (chunks == 1) {                                                                                \
    hipLaunchKernelGGL((rglru_output_kernel<T, true>), grid, dim3(256), 0, s, gates, gate_bias, lam, \
                       (const T*)u, ld_u, (const T*)y, ld_y, y_bias, C, state, carry, chunks,       \
                       (T*)out, ld_out, out_mb, b->seg_start, b->seg_slot, b->seg_pos);             \
  } else {                                                                                          \
    hipLaunchKernelGGL((rglru_local_kernel<T>), grid, dim3(256), 0, s, gates, gate_bias, lam,       \
                       (const T*)u, ld_u, C, carry, chunks, b->seg_start);                          \
    hipLaunchKernelGGL((rglru_output_kernel<T, false>), grid, dim3(256), 0, s, gates, gate_bias,    \
                       lam, (const T*)u, ld_u, (const T*)y, ld_y, y_bias, C, state, carry, chunks,  \
                       (T*)out, ld_out, out_mb, b->seg_start, b->seg_slot, b->seg_pos);             \
    hipLaunchKernelGGL(rglru_state_kernel, dim3((C + 255) / 256, b->nseg), dim3(256), 0, s, C,      \
                       state, carry, chunks, b->seg_start, b->seg_slot, b->seg_pos);                \
  }
  if (dtype == MSA_BF16) {
    RG_RUN(bf16_t)
  } else {
    RG_RUN(float)
  }
#undef RG_RUN
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_delta_scan(const msa_delta_args* a, const msa_batch* b, void* stream) {
  const char* name = "msa_delta_scan";
  int rc = check_delta(name, a, b);
  if (rc) return rc;
  MSA_REQUIRE(a->o, MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  if (a->dtype == MSA_BF16)
    dispatch_delta<bf16_t>(*a, b, false, (hipStream_t)stream);
  else
    dispatch_delta<float>(*a, b, false, (hipStream_t)stream);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_delta_output(const msa_delta_args* a, int M, void* stream) {
  const char* name = "msa_delta_output";
  MSA_REQUIRE(a && a->o && a->gate && a->w && a->out && M > 0 && a->heads > 0 && a->vp > 0 &&
                  a->vp <= 512 && a->vdim <= a->vp,
              MSA_ERR_INVALID_ARG, "%s: bad arguments", name);
  const dim3 grid((unsigned)(((int64_t)M * a->heads + 3) / 4));
  hipStream_t s = (hipStream_t)stream;
  if (a->dtype == MSA_BF16)
    hipLaunchKernelGGL(delta_output_kernel<bf16_t>, grid, dim3(256), 0, s, a->o, (const bf16_t*)a->gate,
                       a->ld_gate, a->gate_act, a->w, a->heads, a->vdim, a->vp, a->eps,
                       (bf16_t*)a->out, a->ld_out, a->out_mb, M);
  else
    hipLaunchKernelGGL(delta_output_kernel<float>, grid, dim3(256), 0, s, a->o, (const float*)a->gate,
                       a->ld_gate, a->gate_act, a->w, a->heads, a->vdim, a->vp, a->eps,
                       (float*)a->out, a->ld_out, 0, M);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}
