// Routing of a mixture of experts: scores, group-limited top-k choice, and the sort of the (token,
// choice) pairs by expert into row tiles for the grouped products.
#include <math.h>

#include "common.h"

namespace {

constexpr int RT_EPL = 8;  // experts per lane: at most 512

// one wave per token; lane l holds experts l, l + 64, ...
__global__ __launch_bounds__(256) void moe_route_kernel(const float* __restrict__ z, int ldz, int M,
                                                        int E, int n_groups, int keep, int top,
                                                        float scale, int32_t* __restrict__ ids,
                                                        float* __restrict__ weights,
                                                        float* __restrict__ shared_gate) {
  const int lane = threadIdx.x & 63;
  const int m = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (m >= M) return;  // wave-uniform
  const float* row = z + (int64_t)m * ldz;
  float s[RT_EPL];
  float mx = -INFINITY;
#pragma unroll
  for (int i = 0; i < RT_EPL; ++i) {
    const int e = lane + 64 * i;
    s[i] = e < E ? row[e] : -INFINITY;
    mx = fmaxf(mx, s[i]);
  }
  mx = wave_max(mx);
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < RT_EPL; ++i) {
    s[i] = lane + 64 * i < E ? expf(s[i] - mx) : 0.f;
    sum += s[i];
  }
  sum = wave_sum(sum);
#pragma unroll
  for (int i = 0; i < RT_EPL; ++i) s[i] /= sum;
  // largest eligible value with the lowest index; a taken one becomes -1 (so that any row, a NaN
  // row included, yields valid ids)
  auto best_of = [&](const float(&v)[RT_EPL], float& bv, int& bi) {
    bv = -2.f, bi = 0;
#pragma unroll
    for (int i = 0; i < RT_EPL; ++i)
      if (lane + 64 * i < E && v[i] > bv) bv = v[i], bi = lane + 64 * i;
    const float best = wave_max(bv);
    unsigned long long at = __ballot(bv == best);
    int id = E - 1;  // (a row of NaN: no lane compares equal)
    for (; at; at &= at - 1)  // one lane, but for ties
      id = min(id, __builtin_amdgcn_readlane(bi, __builtin_ctzll(at)));
    bv = best, bi = id;
  };
  float v[RT_EPL];  // candidates
  if (keep < n_groups) {
    // repeatedly the group of the best remaining expert: `keep` rounds
    const int size = E / n_groups;
    float left[RT_EPL];
#pragma unroll
    for (int i = 0; i < RT_EPL; ++i) left[i] = s[i], v[i] = -1.f;
    for (int k = 0; k < keep; ++k) {
      float bv;
      int bi;
      best_of(left, bv, bi);
      const int g = bi / size;
#pragma unroll
      for (int i = 0; i < RT_EPL; ++i)
        if (lane + 64 * i < E && (lane + 64 * i) / size == g) v[i] = s[i], left[i] = -1.f;
    }
  } else {
#pragma unroll
    for (int i = 0; i < RT_EPL; ++i) v[i] = s[i];
  }
  for (int k = 0; k < top; ++k) {
    float bv;
    int bi;
    best_of(v, bv, bi);
#pragma unroll
    for (int i = 0; i < RT_EPL; ++i)
      if (lane + 64 * i == bi) v[i] = -1.f;
    if (lane == 0) {
      ids[(int64_t)m * top + k] = bi;
      weights[(int64_t)m * top + k] = bv * scale;
    }
  }
  if (shared_gate && lane == 0) shared_gate[m] = sigmoidf(row[E]);
}

// One workgroup per expert: counts all pairs, then writes its own expert's rows in pair order.
__global__ __launch_bounds__(256) void moe_plan_kernel(const int32_t* __restrict__ ids, int P, int E,
                                                       int tile_rows, int32_t* __restrict__ perm,
                                                       int32_t* __restrict__ inverse,
                                                       int32_t* __restrict__ group_end,
                                                       int32_t* __restrict__ tile_group,
                                                       int32_t* __restrict__ tile_row,
                                                       int32_t* __restrict__ n_tiles,
                                                       int max_tiles) {
  __shared__ int hist[512];
  __shared__ int sh_row, sh_tile, wcount[4];
  const int e = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  for (int i = tid; i < E; i += 256) hist[i] = 0;
  __syncthreads();
  for (int p = tid; p < P; p += 256) atomicAdd(&hist[ids[p]], 1);
  __syncthreads();
  if (tid == 0) {
    int row = 0, tile = 0;
    for (int i = 0; i < e; ++i) {
      row += hist[i];
      tile += (hist[i] + tile_rows - 1) / tile_rows;
    }
    sh_row = row;
    sh_tile = tile;
    group_end[e] = row + hist[e];
    if (e == E - 1) *n_tiles = min(max_tiles, tile + (hist[e] + tile_rows - 1) / tile_rows);
  }
  __syncthreads();
  const int mine = hist[e], row0 = sh_row, tile0 = sh_tile;
  for (int t = tid; t < (mine + tile_rows - 1) / tile_rows; t += 256)
    if (tile0 + t < max_tiles) {
      tile_group[tile0 + t] = e;
      tile_row[tile0 + t] = row0 + t * tile_rows;
    }
  int at = row0;
  for (int p0 = 0; p0 < P; p0 += 256) {
    const int p = p0 + tid;
    const bool hit = p < P && ids[p] == e;
    const unsigned long long b = __ballot(hit);
    if (lane == 0) wcount[wave] = __popcll(b);
    __syncthreads();
    int before = at + __popcll(b & ((1ull << lane) - 1));
    int total = 0;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      if (w < wave) before += wcount[w];
      total += wcount[w];
    }
    if (hit) {
      perm[before] = p;
      inverse[p] = before;
    }
    at += total;
    __syncthreads();
  }
}

}  // namespace

extern "C" int msa_moe_route(const float* z, int ldz, int M, int E, int n_groups, int keep, int top,
                             float scale, int32_t* ids, float* weights, float* shared_gate,
                             void* stream) {
  const char* name = "msa_moe_route";
  MSA_REQUIRE(z && ids && weights, MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  MSA_REQUIRE(M >= 0 && E > 0 && E <= 64 * RT_EPL && ldz >= E + (shared_gate ? 1 : 0) && top > 0,
              MSA_ERR_INVALID_ARG, "%s: M=%d E=%d (at most %d) ldz=%d top=%d", name, M, E,
              64 * RT_EPL, ldz, top);
  MSA_REQUIRE(n_groups > 0 && E % n_groups == 0 && keep > 0 && keep <= n_groups &&
                  top <= E / n_groups * keep,
              MSA_ERR_INVALID_ARG, "%s: %d of %d groups over %d experts, top %d", name, keep,
              n_groups, E, top);
  if (M == 0) return MSA_OK;
  hipLaunchKernelGGL(moe_route_kernel, dim3((M + 3) / 4), dim3(256), 0, (hipStream_t)stream, z, ldz, M,
                     E, n_groups, keep, top, scale, ids, weights, shared_gate);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_moe_plan(const int32_t* ids, int P, int E, int tile_rows, int32_t* perm,
                            int32_t* inverse, int32_t* group_end, int32_t* tile_group,
                            int32_t* tile_row, int32_t* n_tiles, int max_tiles, void* stream) {
  const char* name = "msa_moe_plan";
  MSA_REQUIRE(ids && perm && inverse && group_end && tile_group && tile_row && n_tiles,
              MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  MSA_REQUIRE(P > 0 && E > 0 && E <= 512 && tile_rows > 0 &&
                  max_tiles >= P / tile_rows + (E < P ? E : P),
              MSA_ERR_INVALID_ARG, "%s: P=%d E=%d tile_rows=%d max_tiles=%d", name, P, E, tile_rows,
              max_tiles);
  hipLaunchKernelGGL(moe_plan_kernel, dim3(E), dim3(256), 0, (hipStream_t)stream, ids, P, E,
                     tile_rows, perm, inverse, group_end, tile_group, tile_row, n_tiles, max_tiles);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}
