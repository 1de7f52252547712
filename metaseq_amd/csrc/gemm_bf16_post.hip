// bf16 linear layers with a bias, an activation, a second output or decays (msa_linear; kernels:
// gemm_kernels.h).
#include "gemm_kernels.h"

// msa_linear with bf16 operands
int msa_launch_linear_post(const msa_linear_args& a, hipStream_t s) {
  const char* name = "msa_linear";
  int rc = check_linear_args(name, a.x, a.W, a.y ? a.y : (void*)a.y32, a.M, a.N, a.K, false, a.flags,
                             MSA_IN_PACKED | MSA_OUT_PACKED | MSA_OUT2_PACKED);
  if (rc) return rc;
  // packed outputs are produced from packed input only: the row-major kernels store rows
  MSA_REQUIRE(!(a.flags & (MSA_OUT_PACKED | MSA_OUT2_PACKED)) || (a.flags & MSA_IN_PACKED) || a.M <= 64,
              MSA_ERR_INVALID_ARG, "%s: packed output of %lld row-major rows", name, (long long)a.M);
  Epilogue e{};
  e.N = a.N;
  e.n32 = a.n32;
  e.yb = (bf16_t*)a.y;
  e.y32 = a.y32;
  e.n2 = a.y2 ? a.n2 : a.n32;
  e.ldy = e.n2;
  e.ld2 = a.n32 - e.n2;
  e.y2 = (bf16_t*)a.y2;
  e.out_mb = (a.flags & MSA_OUT_PACKED) ? packed_row_blocks(a.M) : 0;
  e.out2_mb = (a.flags & MSA_OUT2_PACKED) ? packed_row_blocks(a.M) : 0;
  e.bias32 = a.bias;
  e.act = a.act;
  e.decay_rate = a.decay_rate;
  e.glu = MSA_GLU_NONE;
  run_linear<MODE_BF_POST>(a.x, a.W, e, a.M, a.N, a.K, a.flags, s);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}
