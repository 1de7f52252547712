// Entry points of the bf16 matrix products (kernels: gemm_kernels.h): linear layers with an optional
// gated activation and fp32 tail columns, and split-K partial sums.
#include "gemm_kernels.h"

namespace {

template <int MODE>
bool run_grouped(const msa_group_linear_args& a, const Epilogue& e, hipStream_t s) {
  static std::atomic<uint64_t> lds_allowed{0};
  auto kernel = linear_quad_kernel<MODE, 8, false, true>;
  if (!allow_lds((const void*)kernel, tq_lds_bytes(8), lds_allowed)) return false;
  const int ncol = (a.N + tq_bn(8) - 1) / tq_bn(8);
  // the shares of the eight XCDs are rounded up: up to 7 workgroups beyond the tiles
  const GroupTiles gt{a.perm, a.tile_group, a.tile_row, a.n_tiles, a.group_end, a.rows_per_x};
  hipLaunchKernelGGL(kernel, dim3(ncol, a.max_tiles + (7 + ncol - 1) / ncol), dim3(TQ_THREADS),
                     tq_lds_bytes(8), s, (const half_t*)a.x, a.W, (int64_t)0, a.N, a.K, 0, 0, 0, e,
                     (float*)nullptr, 0, gt);
  return true;
}

}  // namespace

// Routed products over 256-row tiles (msa_group_linear).  Returns false if the launch is refused.
bool msa_launch_group_quad(const msa_group_linear_args& a, hipStream_t s) {
  Epilogue e{};
  e.N = e.n32 = a.N;
  e.yb = (bf16_t*)a.y;
  e.ldy = (int)a.ldy;
  e.glu = a.glu;
  e.limit = a.limit;
  return a.glu == MSA_GLU_NONE ? run_grouped<MODE_BF>(a, e, s) : run_grouped<MODE_BF_GLU>(a, e, s);
}

extern "C" int msa_linear_bf16(const void* x, const void* W, void* y, float* y32, int64_t M, int N,
                               int K, int n32, int glu, float limit, unsigned flags, void* stream) {
  const char* name = "msa_linear_bf16";
  int rc = check_linear_args(name, x, W, y ? y : (void*)y32, M, N, K, false, flags,
                             MSA_IN_PACKED | MSA_OUT_PACKED);
  if (rc) return rc;
  MSA_REQUIRE(n32 >= 0 && n32 <= N && n32 % (glu == MSA_GLU_NONE ? 16 : 32) == 0,
              MSA_ERR_INVALID_ARG, "%s: n32=%d of N=%d", name, n32, N);
  MSA_REQUIRE((n32 == 0 || y) && (n32 == N || y32), MSA_ERR_INVALID_ARG, "%s: null output", name);
  MSA_REQUIRE(glu >= MSA_GLU_NONE && glu <= MSA_GLU_CLAMPED, MSA_ERR_INVALID_ARG, "%s: glu=%d", name,
              glu);
  // a packed output is produced from packed input only: the row-major kernels store rows
  MSA_REQUIRE(!(flags & MSA_OUT_PACKED) || (flags & MSA_IN_PACKED) || M <= 64, MSA_ERR_INVALID_ARG,
              "%s: packed output of %lld row-major rows", name, (long long)M);
  if (M == 0) return MSA_OK;
  Epilogue e{};
  e.N = N;
  e.n32 = n32;
  e.yb = (bf16_t*)y;
  e.y32 = y32;
  e.ldy = glu == MSA_GLU_NONE ? n32 : n32 / 2;
  e.glu = glu;
  e.limit = limit;
  e.out_mb = (flags & MSA_OUT_PACKED) ? packed_row_blocks(M) : 0;
  if (glu == MSA_GLU_NONE)
    run_linear<MODE_BF>(x, W, e, M, N, K, flags, (hipStream_t)stream);
  else
    run_linear<MODE_BF_GLU>(x, W, e, M, N, K, flags, (hipStream_t)stream);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

extern "C" int msa_linear_bf16_splits(int64_t M, int N, int K, int packed) {
  return packed ? pick_splits(M, N, K, 2) : pick_row_splits(M, N, K);
}

extern "C" int msa_linear_partial_bf16(const void* x, const void* W, float* part, int64_t M, int N,
                                       int K, int S, unsigned flags, void* stream) {
  const char* name = "msa_linear_partial_bf16";
  int rc = check_linear_args(name, x, W, part, M, N, K, false, flags, MSA_IN_PACKED);
  if (rc) return rc;
  MSA_REQUIRE(M >= 1, MSA_ERR_INVALID_ARG, "%s: M=%lld", name, (long long)M);
  if (!(flags & MSA_IN_PACKED)) {
    MSA_REQUIRE(S >= 1 && K % (64 * S) == 0 && K / S >= 128, MSA_ERR_INVALID_ARG,
                "%s: row-major activations need K=%d cut by S=%d into ranges that are multiples "
                "of 64 and at least 128", name, K, S);
    launch_quad_partial<MODE_BF>(x, W, part, M, N, K, S, (hipStream_t)stream);
    MSA_CHECK_LAUNCH(name);
    return MSA_OK;
  }
  const int nks = K / 32, per = (nks + S - 1) / (S > 0 ? S : 1);
  MSA_REQUIRE(S >= 1 && S <= nks && (int64_t)(S - 1) * per < nks, MSA_ERR_INVALID_ARG,
              "%s: S=%d leaves a K range of %d steps empty", name, S, nks);
  Epilogue e{};
  launch_stream<false, MODE_BF>(x, W, nullptr, part, S, (int)M, N, K, e, (hipStream_t)stream);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}
