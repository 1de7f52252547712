// Grouped matrix products: block-diagonal layers, per-head projections and routed experts.
//
// bf16: a workgroup of four waves owns MT x 16 rows of one group and a range of 16-column tiles.
// Weights come straight from the tile-packed layout in memory (one KB per wave instruction), the
// activation fragments straight from the rows (16 bytes per lane; rows may be gathered through a
// permutation, and may lie in the packed activation layout), so there is no LDS staging and no
// barrier in the main loop.  Few rows (a decode step): the four waves split K and their sums meet
// in LDS; many rows: every wave owns its own column tiles.  Loads run one stage ahead of the MFMAs.
//
// Routed products with more than 64 rows per expert run on the four-wave 256 x 256 kernel of the dense
// products instead (gemm_kernels.h).
//
// fp32: 64 x 64 tiles through LDS on the vector ALU in full fp32; also the fp32 linear layers.
#include <math.h>

#include "common.h"

namespace {

struct Rows {  // the rows a workgroup works on
  int group;
  int64_t first, end;  // of y (and of x unless permuted)
};

__device__ __forceinline__ bool find_rows(const msa_group_linear_args& a, int row_tile, int z,
                                          Rows& r) {
  if (a.tile_group) {
    if (row_tile >= *a.n_tiles) return false;
    r.group = a.tile_group[row_tile];
    r.first = a.tile_row[row_tile];
    const int64_t ge = a.group_end[r.group];
    r.end = r.first + a.tile_rows < ge ? r.first + a.tile_rows : ge;
  } else {
    r.group = z;
    r.first = (int64_t)row_tile * a.tile_rows;
    r.end = r.first + a.tile_rows < a.M ? r.first + a.tile_rows : a.M;
  }
  return r.first < r.end;
}

template <bool GLU>
__device__ __forceinline__ void store4(const msa_group_linear_args& a, int group, int64_t row, int n,
                                       float4_t v) {
  row += a.y_row0;
  if constexpr (GLU) {
    const float o0 = glu_act(a.glu, v[0], v[1], a.limit), o1 = glu_act(a.glu, v[2], v[3], a.limit);
    const int c = group * a.y_group + (n >> 1);
    if (a.y_f32) {
      float* y = (float*)a.y + row * a.ldy + c;
      y[0] = o0, y[1] = o1;
    } else {
      bf16_t* y = (bf16_t*)a.y + (a.y_mb > 0 ? packed_act_offset((int)row, c, a.y_mb)
                                             : row * a.ldy + c);
      *reinterpret_cast<bf16x2_t*>(y) = bf16x2_t{(bf16_t)o0, (bf16_t)o1};
    }
  } else {
    const int c = group * a.y_group + n;
    if (a.y_f32) {
      *reinterpret_cast<float4_t*>((float*)a.y + row * a.ldy + c) = v;
    } else {
      bf16_t* y = (bf16_t*)a.y + (a.y_mb > 0 ? packed_act_offset((int)row, c, a.y_mb)
                                             : row * a.ldy + c);
      *reinterpret_cast<bf16x4_t*>(y) =
          bf16x4_t{(bf16_t)v[0], (bf16_t)v[1], (bf16_t)v[2], (bf16_t)v[3]};
    }
  }
}

// MT row blocks of 16 per workgroup, NT column tiles per wave, KW waves share a column range and
// split K, U 32-wide steps per stage.
template <int MT, int NT, int KW, int U, bool GLU>
__global__ __launch_bounds__(256) void group_linear_bf16_kernel(msa_group_linear_args a) {
  constexpr int NW = 4 / KW;  // waves side by side over the columns
  __shared__ float4_t red[KW > 1 ? KW : 1][KW > 1 ? NW * MT * NT : 1][64];
  Rows rw;
  if (!find_rows(a, blockIdx.y, blockIdx.z, rw)) return;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int kw = wave % KW, nw = wave / KW;
  const int nks = a.K >> 5, ntiles = a.N >> 4;
  const int t0 = (blockIdx.x * NW + nw) * NT;
  const bf16_t* Wg = (const bf16_t*)a.W + (int64_t)rw.group * a.N * a.K;
  const bf16_t* wp[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j)
    wp[j] = Wg + (int64_t)min(t0 + j, ntiles - 1) * nks * 512 + lane * 8;
  const int xg = a.x_groups > 0 ? rw.group % a.x_groups : rw.group;
  const bf16_t* xp[MT];
  const int64_t kstep = a.x_mb > 0 ? (int64_t)a.x_mb * 512 : 32;
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    int64_t r = rw.first + i * 16 + (lane & 15);
    if (r >= rw.end) r = rw.end - 1;
    const int64_t m = a.perm ? a.perm[r] / a.rows_per_x : r;
    if (a.x_mb > 0)
      xp[i] = (const bf16_t*)a.x +
              ((m >> 4) * 64 + (lane & 48) + (m & 15)) * 8 + (int64_t)xg * a.x_group;
    else
      xp[i] = (const bf16_t*)a.x + m * a.ldx + (int64_t)xg * a.x_group + (lane >> 4) * 8;
  }
  struct Stage {
    half8_t w[U][NT], x[U][MT];
  };
  Stage s[2];
  const int nst = (nks + KW * U - 1) / (KW * U);
  auto load = [&](Stage& st, int idx) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int ks = min((idx * U + u) * KW + kw, nks - 1);
#pragma unroll
      for (int j = 0; j < NT; ++j)
        st.w[u][j] = *reinterpret_cast<const half8_t*>(wp[j] + (int64_t)ks * 512);
#pragma unroll
      for (int i = 0; i < MT; ++i)
        st.x[u][i] = *reinterpret_cast<const half8_t*>(xp[i] + ks * kstep);
    }
  };
  float4_t acc[MT][NT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[i][j] = float4_t{0.f, 0.f, 0.f, 0.f};
  auto mma = [&](Stage& st, int idx) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if ((idx * U + u) * KW + kw >= nks) break;  // wave-uniform
#pragma unroll
      for (int i = 0; i < MT; ++i)
#pragma unroll
        for (int j = 0; j < NT; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              __builtin_bit_cast(bf16x8_t, st.w[u][j]), __builtin_bit_cast(bf16x8_t, st.x[u][i]),
              acc[i][j], 0, 0, 0);
    }
  };
  load(s[0], 0);
  int idx = 0;
  for (; idx + 2 <= nst; idx += 2) {
    load(s[1], idx + 1);
    mma(s[0], idx);
    load(s[0], idx + 2);  // past the end: a clamped address, never multiplied
    mma(s[1], idx + 1);
  }
  if (idx < nst) mma(s[0], idx);

  // a lane holds row lane % 16 of every row block, columns 4 * (lane / 16) .. + 3 of every tile
  if constexpr (KW > 1) {
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int j = 0; j < NT; ++j) red[kw][(nw * MT + i) * NT + j][lane] = acc[i][j];
    __syncthreads();
    for (int e = threadIdx.x; e < NW * MT * NT * 64; e += 256) {
      const int t = e >> 6, l = e & 63;
      const int j = t % NT, i = (t / NT) % MT, w = t / (NT * MT);
      float4_t v = red[0][t][l];
#pragma unroll
      for (int k = 1; k < KW; ++k) v += red[k][t][l];
      const int64_t r = rw.first + i * 16 + (l & 15);
      const int tile = (blockIdx.x * NW + w) * NT + j;
      if (r < rw.end && tile < ntiles)
        store4<GLU>(a, rw.group, r, tile * 16 + ((l >> 4) << 2), v);
    }
  } else {
#pragma unroll
    for (int i = 0; i < MT; ++i) {
      const int64_t r = rw.first + i * 16 + (lane & 15);
#pragma unroll
      for (int j = 0; j < NT; ++j)
        if (r < rw.end && t0 + j < ntiles)
          store4<GLU>(a, rw.group, r, (t0 + j) * 16 + ((lane >> 4) << 2), acc[i][j]);
    }
  }
}

template <int MT, int NT, int KW, int U>
void launch_bf16(const msa_group_linear_args& a, int row_tiles, hipStream_t s) {
  constexpr int NB = 4 / KW * NT;
  const dim3 grid((a.N / 16 + NB - 1) / NB, row_tiles, a.tile_group ? 1 : a.groups);
  if (a.glu == MSA_GLU_NONE)
    hipLaunchKernelGGL((group_linear_bf16_kernel<MT, NT, KW, U, false>), grid, dim3(256), 0, s, a);
  else
    hipLaunchKernelGGL((group_linear_bf16_kernel<MT, NT, KW, U, true>), grid, dim3(256), 0, s, a);
}

// ---- fp32 -----------------------------------------------------------------------------------
// 64 rows x 64 columns per workgroup, 16-wide K stages through LDS, 4 x 4 outputs per thread.
// n32 splits the columns between y and y32 (linear layers); glu pairs lie within a thread.
// `post` (linear layers only): bias, activation, second output and decays as in MODE_BF_POST.
struct PostF32 {
  const float *bias, *decay_rate;
  float* y2;
  int act, n2, used;
};

__global__ __launch_bounds__(256) void linear_f32_kernel(msa_group_linear_args a, float* y32, int n32,
                                                         PostF32 post) {
  __shared__ float lx[16][64 + 4], lw[16][64 + 4];
  Rows rw;
  if (!find_rows(a, blockIdx.y, blockIdx.z, rw)) return;
  const int tid = threadIdx.x, n0 = blockIdx.x * 64;
  const float* Wg = (const float*)a.W + (int64_t)rw.group * a.N * a.K;
  const int tr = tid >> 4, tc = tid & 15;  // rows 4 tr .., columns 4 tc ..
  const int lr = tid >> 2, lk = (tid & 3) * 4;  // staging: row lr, K offset lk
  int64_t r = rw.first + lr;
  if (r >= rw.end) r = rw.end - 1;
  const int64_t m = a.perm ? a.perm[r] / a.rows_per_x : r;
  const int xg = a.x_groups > 0 ? rw.group % a.x_groups : rw.group;
  const float* xr = (const float*)a.x + m * a.ldx + (int64_t)xg * a.x_group;
  const float* wr = Wg + (int64_t)min(n0 + lr, a.N - 1) * a.K;
  float acc[4][4] = {};
  for (int k0 = 0; k0 < a.K; k0 += 16) {
    const float4_t xv = *reinterpret_cast<const float4_t*>(xr + k0 + lk);
    const float4_t wv = *reinterpret_cast<const float4_t*>(wr + k0 + lk);
#pragma unroll
    for (int i = 0; i < 4; ++i) lx[lk + i][lr] = xv[i], lw[lk + i][lr] = wv[i];
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 16; ++k) {
      const float4_t xk = *reinterpret_cast<const float4_t*>(&lx[k][tr * 4]);
      const float4_t wk = *reinterpret_cast<const float4_t*>(&lw[k][tc * 4]);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(xk[i], wk[j], acc[i][j]);
    }
    __syncthreads();
  }
  const int n = n0 + tc * 4;
  if (n >= a.N) return;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int64_t row = rw.first + tr * 4 + i;
    if (row >= rw.end) break;
    float4_t v = {acc[i][0], acc[i][1], acc[i][2], acc[i][3]};
    if (post.used) {
      if (post.bias) v += *reinterpret_cast<const float4_t*>(post.bias + n);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (n < n32)
          v[j] = post.act == MSA_ACT_RELU2 ? relu2(v[j]) : v[j];
        else if (post.decay_rate)
          v[j] = decay_of(v[j], post.decay_rate[n - n32 + j]);
      if (n < n32 && n >= post.n2) {
        *reinterpret_cast<float4_t*>(post.y2 + row * (n32 - post.n2) + (n - post.n2)) = v;
        continue;
      }
    }
    if (n >= n32)
      *reinterpret_cast<float4_t*>(y32 + row * (a.N - n32) + (n - n32)) = v;
    else if (a.glu == MSA_GLU_NONE)
      store4<false>(a, rw.group, row, n, v);
    else
      store4<true>(a, rw.group, row, n, v);
  }
}

}  // namespace

extern "C" int msa_group_linear(const msa_group_linear_args* args, void* stream) {
  const char* name = "msa_group_linear";
  MSA_REQUIRE(args && args->x && args->W && args->y, MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  msa_group_linear_args a = *args;
  MSA_REQUIRE(a.dtype == MSA_BF16 || a.dtype == MSA_F32, MSA_ERR_INVALID_ARG, "%s: dtype", name);
  MSA_REQUIRE(a.N > 0 && a.N % 16 == 0 && a.K > 0 && a.K % 32 == 0 && a.groups > 0,
              MSA_ERR_INVALID_ARG, "%s: N=%d K=%d groups=%d", name, a.N, a.K, a.groups);
  MSA_REQUIRE(a.ldx % 8 == 0 && a.x_group % 8 == 0 && a.ldy % 4 == 0 && a.y_group % 4 == 0,
              MSA_ERR_INVALID_ARG, "%s: strides", name);
  MSA_REQUIRE(a.dtype == MSA_BF16 || (a.x_mb == 0 && a.y_mb == 0), MSA_ERR_INVALID_ARG,
              "%s: fp32 activations are row-major", name);
  MSA_REQUIRE(a.x_mb == 0 || a.x_group == 0, MSA_ERR_INVALID_ARG,
              "%s: packed activations have no column groups", name);
  const bool routed = a.tile_group != nullptr;
  MSA_REQUIRE(!routed || (a.tile_row && a.n_tiles && a.group_end && a.max_tiles > 0 &&
                          a.tile_rows > 0 && (a.tile_rows <= 64 || a.tile_rows == 256) && (!a.perm || a.rows_per_x > 0)),
              MSA_ERR_INVALID_ARG, "%s: incomplete routing tables", name);
  MSA_REQUIRE(routed || !a.perm, MSA_ERR_INVALID_ARG, "%s: a permutation needs tiles", name);
  if (!routed && a.M <= 0) return MSA_OK;
  if (a.dtype == MSA_F32) a.y_f32 = 1;
  hipStream_t s = (hipStream_t)stream;
  int rows = a.tile_rows;
  if (!routed) a.tile_rows = rows = a.dtype == MSA_F32 ? 64 : a.M <= 16 ? 16 : a.M <= 32 ? 32 : 64;
  const int64_t row_tiles = routed ? a.max_tiles : (a.M + rows - 1) / rows;
  MSA_REQUIRE(row_tiles <= 65535, MSA_ERR_INVALID_ARG, "%s: too many rows", name);
  if (rows == 256) {
    MSA_REQUIRE(a.dtype == MSA_BF16 && a.x_mb == 0 && a.y_mb == 0 && !a.y_f32 && a.ldx == a.K &&
                    a.K % 64 == 0 && a.K >= 128 && a.y_row0 == 0 && a.M * a.K * 2 < (1ll << 32) &&
                    (a.glu == MSA_GLU_NONE || a.N % 32 == 0),
                MSA_ERR_INVALID_ARG, "%s: 256-row tiles of row-major bf16 rows, K=%d", name, a.K);
    MSA_REQUIRE(msa_launch_group_quad(a, s), MSA_ERR_HIP, "%s: LDS limit", name);
  } else if (a.dtype == MSA_F32) {
    hipLaunchKernelGGL(linear_f32_kernel, dim3((a.N + 63) / 64, (unsigned)row_tiles,
                                               routed ? 1 : a.groups),
                       dim3(256), 0, s, a, (float*)nullptr, a.N, PostF32{});
  } else if (rows <= 16) {
    launch_bf16<1, 2, 4, 4>(a, (int)row_tiles, s);
  } else if (rows <= 32) {
    launch_bf16<2, 2, 4, 2>(a, (int)row_tiles, s);
  } else if (a.N <= 128 || (!routed && a.M <= 128)) {
    launch_bf16<4, 2, 2, 1>(a, (int)row_tiles, s);
  } else {
    launch_bf16<4, 4, 1, 1>(a, (int)row_tiles, s);
  }
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_linear_f32(const float* x, const float* W, float* y, float* y32, int64_t M, int N,
                              int K, int n32, int glu, float limit, void* stream) {
  const char* name = "msa_linear_f32";
  MSA_REQUIRE(x && W && (y || n32 == 0) && (y32 || n32 == N), MSA_ERR_INVALID_ARG,
              "%s: null pointer", name);
  MSA_REQUIRE(M >= 0 && N > 0 && N % 16 == 0 && K > 0 && K % 32 == 0 && n32 >= 0 && n32 <= N &&
                  n32 % 4 == 0 && (M + 63) / 64 <= 65535,
              MSA_ERR_INVALID_ARG, "%s: M=%lld N=%d K=%d n32=%d", name, (long long)M, N, K, n32);
  if (M == 0) return MSA_OK;
  msa_group_linear_args a{};
  a.dtype = MSA_F32;
  a.x = x;
  a.ldx = K;
  a.W = W;
  a.y = y;
  a.ldy = glu == MSA_GLU_NONE ? n32 : n32 / 2;
  a.y_f32 = 1;
  a.N = N;
  a.K = K;
  a.groups = 1;
  a.glu = glu;
  a.limit = limit;
  a.M = M;
  a.tile_rows = 64;
  hipLaunchKernelGGL(linear_f32_kernel, dim3((N + 63) / 64, (unsigned)((M + 63) / 64), 1), dim3(256),
                     0, (hipStream_t)stream, a, y32, n32, PostF32{});
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_linear(const msa_linear_args* args, void* stream) {
  const char* name = "msa_linear";
  MSA_REQUIRE(args && args->x && args->W, MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  const msa_linear_args& p = *args;
  MSA_REQUIRE(p.dtype == MSA_BF16 || p.dtype == MSA_F32, MSA_ERR_INVALID_ARG, "%s: dtype", name);
  MSA_REQUIRE(p.M >= 0 && p.N > 0 && p.N % 16 == 0 && p.K > 0 && p.K % 64 == 0 && p.n32 >= 0 &&
                  p.n32 <= p.N && p.n32 % 16 == 0 && (p.M + 63) / 64 <= 65535 &&
                  (!p.y2 || (p.n2 >= 0 && p.n2 <= p.n32 && p.n2 % 16 == 0)),
              MSA_ERR_INVALID_ARG, "%s: M=%lld N=%d K=%d n32=%d n2=%d", name, (long long)p.M, p.N, p.K,
              p.n32, p.n2);
  const int n2 = p.y2 ? p.n2 : p.n32;
  MSA_REQUIRE((p.y || n2 == 0) && (p.y32 || p.n32 == p.N), MSA_ERR_INVALID_ARG, "%s: null output", name);
  MSA_REQUIRE(p.act == MSA_ACT_NONE || p.act == MSA_ACT_RELU2, MSA_ERR_INVALID_ARG, "%s: act=%d", name,
              p.act);
  if (p.M == 0) return MSA_OK;
  if (p.dtype == MSA_BF16) return msa_launch_linear_post(p, (hipStream_t)stream);
  MSA_REQUIRE(p.flags == 0, MSA_ERR_INVALID_ARG, "%s: fp32 activations are row-major", name);
  msa_group_linear_args a{};
  a.dtype = MSA_F32;
  a.x = p.x;
  a.ldx = p.K;
  a.W = p.W;
  a.y = p.y;
  a.ldy = n2;
  a.y_f32 = 1;
  a.N = p.N;
  a.K = p.K;
  a.groups = 1;
  a.glu = MSA_GLU_NONE;
  a.M = p.M;
  a.tile_rows = 64;
  const PostF32 post{p.bias, p.decay_rate, (float*)p.y2, p.act, n2, 1};
  hipLaunchKernelGGL(linear_f32_kernel, dim3((p.N + 63) / 64, (unsigned)((p.M + 63) / 64), 1), dim3(256),
                     0, (hipStream_t)stream, a, p.y32, p.n32, post);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}
