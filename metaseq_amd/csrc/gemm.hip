// Entry points of the fp16 / int8 matrix products (kernels: gemm_kernels.h): weight packing,
// linear layers, split-K partial sums, the QKV projection and the fused vocabulary projection.
#include "gemm_kernels.h"

namespace {

// ---- weight packing ---------------------------------------------------------------------
// fp16: block (tile t = n/16, step ks = k/32) at halves ((t * K/32 + ks) * 512); inside the block
// lane l = 16*((k%32)/8) + n%16 owns halves l*8 .. l*8+7 = W[n][8*(k/8) .. +7].
// int8: block (t, ks8 = k/64) at bytes ((t * K/64 + ks8) * 1024); lane l = 16*g + r owns 16 bytes:
// bytes 0..7 = W[16t+r][64*ks8 + 8g .. +7] and bytes 8..15 = W[16t+r][64*ks8 + 32 + 8g .. +7],
// i.e. the A fragments of the two 32-wide steps the block covers; every byte is stored as
// q + 128.
__global__ __launch_bounds__(256) void pack_f16_kernel(const half_t* __restrict__ src,
                                                       half_t* __restrict__ dst, int N, int K,
                                                       bool unpack) {
  const int64_t piece = (int64_t)blockIdx.x * 256 + threadIdx.x;  // one 16-byte piece
  const int nks = K >> 5;
  if (piece >= (int64_t)N * K / 8) return;
  const int lane = (int)(piece & 63);
  const int64_t blk = piece >> 6;
  const int ks = (int)(blk % nks), t = (int)(blk / nks);
  const int64_t rm = ((int64_t)t * 16 + (lane & 15)) * K + ks * 32 + (lane >> 4) * 8;
  if (unpack)
    *reinterpret_cast<half8_t*>(dst + rm) = *reinterpret_cast<const half8_t*>(src + piece * 8);
  else
    *reinterpret_cast<half8_t*>(dst + piece * 8) = *reinterpret_cast<const half8_t*>(src + rm);
}

__global__ __launch_bounds__(256) void pack_i8_kernel(const int8_t* __restrict__ src,
                                                      int8_t* __restrict__ dst, int N, int K,
                                                      bool unpack) {
  const int64_t piece = (int64_t)blockIdx.x * 256 + threadIdx.x;  // one 8-byte piece
  const int nks8 = K >> 6;
  if (piece >= (int64_t)N * K / 8) return;
  const int half = (int)(piece & 1), lane = (int)((piece >> 1) & 63);
  const int64_t blk = piece >> 7;
  const int ks8 = (int)(blk % nks8), t = (int)(blk / nks8);
  const int64_t rm = ((int64_t)t * 16 + (lane & 15)) * K + ks8 * 64 + half * 32 + (lane >> 4) * 8;
  // packed bytes are q + 128 (the sign bit flipped): the kernels expand them without a
  // sign fix-up
  uint2 v = *reinterpret_cast<const uint2*>(unpack ? src + piece * 8 : src + rm);
  v.x ^= 0x80808080u;
  v.y ^= 0x80808080u;
  *reinterpret_cast<uint2*>(unpack ? dst + rm : dst + piece * 8) = v;
}

// packed int8 -> packed fp16, each element round(q * scale): int8 block (t, ks8) becomes the fp16
// blocks (t, 2 ks8) and (t, 2 ks8 + 1), and a lane's bytes 0..7 / 8..15 become its 8 halves in
// the first / second of them (the lane index is the same in both layouts).  One thread per lane
// and int8 block.
__global__ __launch_bounds__(256) void expand_w8_kernel(const uint8_t* __restrict__ Wq,
                                                        const half_t* __restrict__ scales,
                                                        half_t* __restrict__ dst, int N, int K) {
  const int64_t id = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (id >= (int64_t)N * K / 16) return;
  const int lane = (int)(id & 63);
  const int64_t blk = id >> 6;
  const int nks8 = K >> 6;
  const int t = (int)(blk / nks8);
  typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
  const u32x4 v = __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(Wq) + id);
  const half_t sc = scales[t * 16 + (lane & 15)];
  half8_t* out = reinterpret_cast<half8_t*>(dst) + (blk * 2) * 64 + lane;
  out[0] = dequant8(v[0], v[1], sc);
  out[64] = dequant8(v[2], v[3], sc);
}

template <bool W8>
int linear_entry(const char* name, const void* x, const void* W, const void* scales,
                 const void* bias, const void* residual, void* y, int64_t M, int N, int K,
                 unsigned flags, void* stream) {
  int rc = check_linear_args(name, x, W, y, M, N, K, W8, flags,
                             MSA_EPI_RELU | MSA_IN_PACKED | MSA_OUT_PACKED);
  if (rc) return rc;
  MSA_REQUIRE(!W8 || scales, MSA_ERR_INVALID_ARG, "%s: null scales", name);
  MSA_REQUIRE(!((flags & MSA_OUT_PACKED) && residual && residual == y), MSA_ERR_INVALID_ARG,
              "%s: a packed output cannot alias the row-major residual", name);
  if (M == 0) return MSA_OK;
  Epilogue e{};
  e.bias = (const half_t*)bias;
  e.residual = (const half_t*)residual;
  e.y = (half_t*)y;
  e.N = N;
  e.flags = flags & MSA_EPI_RELU;
  e.out_mb = (flags & MSA_OUT_PACKED) ? packed_row_blocks(M) : 0;
  if (flags & MSA_IN_PACKED)
    launch_stream<W8, MODE_PLAIN>(x, W, scales, nullptr, 1, (int)M, N, K, e, (hipStream_t)stream);
  else
    launch_tiled<W8, MODE_PLAIN>(x, W, scales, M, N, K, e, (hipStream_t)stream);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

template <bool W8>
int partial_entry(const char* name, const void* x, const void* W, const void* scales, float* part,
                  int64_t M, int N, int K, int S, unsigned flags, void* stream) {
  int rc = check_linear_args(name, x, W, part, M, N, K, W8, flags, MSA_IN_PACKED);
  if (rc) return rc;
  MSA_REQUIRE(!W8 || scales, MSA_ERR_INVALID_ARG, "%s: null scales", name);
  if (!(flags & MSA_IN_PACKED)) {
    // row-major activations: the MFMA tile kernel over S equal K ranges
    MSA_REQUIRE(!W8, MSA_ERR_INVALID_ARG,
                "%s: partial sums of row-major activations exist for fp16 weights only (expand "
                "the int8 matrix with msa_expand_weight_w8_f16 first)", name);
    MSA_REQUIRE(M >= 1, MSA_ERR_INVALID_ARG, "%s: M=%lld", name, (long long)M);
    MSA_REQUIRE(S >= 1 && K % (64 * S) == 0 && K / S >= 128, MSA_ERR_INVALID_ARG,
                "%s: row-major activations need K=%d cut by S=%d into ranges that are multiples "
                "of 64 and at least 128", name, K, S);
    launch_quad_partial<MODE_PLAIN>(x, W, part, M, N, K, S, (hipStream_t)stream);
    MSA_CHECK_LAUNCH(name);
    return MSA_OK;
  }
  MSA_REQUIRE(M >= 1 && M <= MSA_PACKED_MAX_ROWS, MSA_ERR_INVALID_ARG,
              "%s: packed activations need 1 <= M <= %d (M=%lld)", name, MSA_PACKED_MAX_ROWS,
              (long long)M);
  MSA_REQUIRE(S >= 1 && S <= K / (W8 ? 64 : 32), MSA_ERR_INVALID_ARG,
              "%s: S=%d outside 1..%d", name, S, K / (W8 ? 64 : 32));
  {
    // the ranges are ceil(steps / S) 32-wide steps each (an even count for int8): every one of
    // the S slices must get at least one step, or it would stay unwritten
    const int nks = K / 32;
    int per = (nks + S - 1) / S;
    if (W8) per = (per + 1) & ~1;
    MSA_REQUIRE((int64_t)(S - 1) * per < nks, MSA_ERR_INVALID_ARG,
                "%s: S=%d leaves a K range empty (K=%d is cut into ranges of %d elements)", name, S,
                K, per * 32);
  }
  Epilogue e{};
  launch_stream<W8, MODE_PLAIN>(x, W, scales, part, S, (int)M, N, K, e, (hipStream_t)stream);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

template <bool W8>
int qkv_entry(const char* name, const void* x, const void* W, const void* scales, const void* bqkv,
              void* q_out, void* Kc, void* Vc, int B, int T, int H, int hd, int S0, int S_cap,
              int K, unsigned flags, const int32_t* len_dev, void* stream) {
  MSA_REQUIRE(!len_dev || T == 1, MSA_ERR_INVALID_ARG, "%s: a device-side length needs T == 1",
              name);
  MSA_REQUIRE(q_out && Kc && Vc, MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  MSA_REQUIRE(B > 0 && T > 0 && H > 0 && hd > 0 && hd % 8 == 0 && S0 >= 0, MSA_ERR_INVALID_ARG,
              "%s: bad shape B=%d T=%d H=%d hd=%d S0=%d", name, B, T, H, hd, S0);
  MSA_REQUIRE((int64_t)S0 + T <= S_cap, MSA_ERR_CAPACITY,
              "%s: S0 + T = %d exceeds the cache capacity %d", name, S0 + T, S_cap);
  const int64_t M = (int64_t)B * T;
  const int N = 3 * H * hd;
  int rc = check_linear_args(name, x, W, q_out, M, N, K, W8, flags, MSA_IN_PACKED);
  if (rc) return rc;
  MSA_REQUIRE(!W8 || scales, MSA_ERR_INVALID_ARG, "%s: null scales", name);
  Epilogue e{};
  e.bias = (const half_t*)bqkv;
  e.N = N;
  e.q_out = (half_t*)q_out;
  e.Kc = (half_t*)Kc;
  e.Vc = (half_t*)Vc;
  e.T = T;
  e.H = H;
  e.hd = hd;
  e.hd_shift = (hd & (hd - 1)) == 0 ? __builtin_ctz((unsigned)hd) : -1;
  e.S0 = S0;
  e.len_dev = len_dev;
  e.S_cap = S_cap;
  e.qscale = (float)pow((double)hd, -0.5);  // the reference's head_dim ** -0.5, cast to fp32
  if (flags & MSA_IN_PACKED)
    launch_stream<W8, MODE_QKV>(x, W, scales, nullptr, 1, (int)M, N, K, e, (hipStream_t)stream);
  else
    launch_tiled<W8, MODE_QKV>(x, W, scales, M, N, K, e, (hipStream_t)stream);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

int pack_entry(const char* name, const void* src, void* dst, int N, int K, bool i8, bool unpack,
               void* stream) {
  MSA_REQUIRE(src && dst && src != dst, MSA_ERR_INVALID_ARG, "%s: null or aliased pointers", name);
  MSA_REQUIRE(N > 0 && K > 0 && N % 16 == 0 && K % (i8 ? 64 : 32) == 0, MSA_ERR_INVALID_ARG,
              "%s: N=%d must be a multiple of 16 and K=%d of %d", name, N, K, i8 ? 64 : 32);
  const int64_t pieces = (int64_t)N * K / 8;
  const dim3 grid((unsigned)((pieces + 255) / 256));
  if (i8)
    hipLaunchKernelGGL(pack_i8_kernel, grid, dim3(256), 0, (hipStream_t)stream, (const int8_t*)src,
                       (int8_t*)dst, N, K, unpack);
  else
    hipLaunchKernelGGL(pack_f16_kernel, grid, dim3(256), 0, (hipStream_t)stream,
                       (const half_t*)src, (half_t*)dst, N, K, unpack);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}

}  // namespace

extern "C" int msa_pack_weight_f16(const void* src, void* dst, int N, int K, void* stream) {
  return pack_entry("msa_pack_weight_f16", src, dst, N, K, false, false, stream);
}
extern "C" int msa_unpack_weight_f16(const void* src, void* dst, int N, int K, void* stream) {
  return pack_entry("msa_unpack_weight_f16", src, dst, N, K, false, true, stream);
}
extern "C" int msa_pack_weight_i8(const int8_t* src, int8_t* dst, int N, int K, void* stream) {
  return pack_entry("msa_pack_weight_i8", src, dst, N, K, true, false, stream);
}
extern "C" int msa_unpack_weight_i8(const int8_t* src, int8_t* dst, int N, int K, void* stream) {
  return pack_entry("msa_unpack_weight_i8", src, dst, N, K, true, true, stream);
}

extern "C" int msa_expand_weight_w8_f16(const int8_t* Wq, const void* scales, void* Wp, int N,
                                        int K, void* stream) {
  MSA_REQUIRE(Wq && scales && Wp && (const void*)Wq != Wp, MSA_ERR_INVALID_ARG,
              "msa_expand_weight_w8_f16: null or aliased pointers");
  MSA_REQUIRE(N > 0 && K > 0 && N % 16 == 0 && K % 64 == 0, MSA_ERR_INVALID_ARG,
              "msa_expand_weight_w8_f16: N=%d must be a multiple of 16 and K=%d of 64", N, K);
  const int64_t n = (int64_t)N * K / 16;
  hipLaunchKernelGGL(expand_w8_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0,
                     (hipStream_t)stream, (const uint8_t*)Wq, (const half_t*)scales, (half_t*)Wp,
                     N, K);
  MSA_CHECK_LAUNCH("msa_expand_weight_w8_f16");
  return MSA_OK;
}

extern "C" int64_t msa_lm_head_select_workspace_bytes(int M) {
  // one partial per row and workgroup; the streaming kernel never launches more workgroups
  // than there are compute units
  return (int64_t)(M > 0 ? M : 0) * num_cus() * (int64_t)sizeof(SelectPartial);
}

namespace {
int lm_head_select_impl(const char* name, const void* x, const void* Ep, void* logits,
                        void* workspace, int M, int V, int K, float temperature,
                        const int32_t* banned_host, int n_banned, const int32_t* stop_host,
                        int n_stop, uint8_t* finished, const uint8_t* row_mode, int force_eos_all,
                        int eos_idx, int64_t* tok, int64_t tok_stride, float* score,
                        int64_t score_stride, const int32_t* len_dev, void* stream) {
  MSA_REQUIRE(x && Ep && workspace && tok && score, MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  MSA_REQUIRE(M >= 1 && M <= 64 && V > 0 && V % 16 == 0 && K > 0 && K % 32 == 0,
              MSA_ERR_INVALID_ARG, "%s: bad shape M=%d V=%d K=%d (1 <= M <= 64, V %% 16, K %% 32)",
              name, M, V, K);
  MSA_REQUIRE(n_banned >= 0 && n_banned <= 16 && (n_banned == 0 || banned_host),
              MSA_ERR_INVALID_ARG, "%s: n_banned=%d (0..16)", name, n_banned);
  MSA_REQUIRE(n_stop >= 0 && n_stop <= 15 && (n_stop == 0 || stop_host), MSA_ERR_INVALID_ARG,
              "%s: n_stop=%d (0..15)", name, n_stop);
  MSA_REQUIRE(eos_idx >= 0 && eos_idx < V, MSA_ERR_INVALID_ARG,
              "%s: eos_idx=%d outside the vocabulary", name, eos_idx);
  MSA_REQUIRE(temperature >= 0.f, MSA_ERR_INVALID_ARG, "%s: temperature < 0", name);
  Epilogue e{};
  e.y = (half_t*)logits;
  e.N = V;
  e.partials = (SelectPartial*)workspace;
  e.finished = finished;
  e.row_mode = row_mode;
  e.early.n = 1 + n_stop;
  e.early.id[0] = eos_idx;
  for (int i = 0; i < n_stop; ++i) e.early.id[1 + i] = stop_host[i];
  e.banned.n = n_banned;
  for (int i = 0; i < n_banned; ++i) e.banned.id[i] = banned_host[i];
  e.temperature = temperature;
  e.scale = temperature > 0.f && temperature != 1.0f;
  e.force_eos_all = force_eos_all;
  e.eos = eos_idx;
  IdList stop{};
  stop.n = n_stop;
  for (int i = 0; i < n_stop; ++i) stop.id[i] = stop_host[i];
  // same decomposition as launch_stream_mb at S = 1: the partial stride is its grid size
  const int ntiles = V / 16;
  const int tiles_per_wg = (ntiles + num_cus() - 1) / num_cus();
  const int gx = (ntiles + tiles_per_wg - 1) / tiles_per_wg;
  launch_stream<false, MODE_SELECT>(x, Ep, nullptr, nullptr, 1, M, V, K, e, (hipStream_t)stream);
  MSA_CHECK_LAUNCH(name);
  msa_launch_select_combine((const SelectPartial*)workspace, gx, M, stop, finished, eos_idx, tok,
                            tok_stride, score, score_stride, len_dev, (hipStream_t)stream);
  MSA_CHECK_LAUNCH(name);
  return MSA_OK;
}
}  // namespace

extern "C" int msa_lm_head_greedy_select_f16(
    const void* x, const void* Ep, void* logits, void* workspace, int M, int V, int K,
    float temperature, const int32_t* banned_host, int n_banned, const int32_t* stop_host,
    int n_stop, uint8_t* finished, const uint8_t* row_mode, int force_eos_all, int eos_idx,
    int64_t* tok, int64_t tok_stride, float* score, int64_t score_stride, const int32_t* len_dev,
    void* stream) {
  return lm_head_select_impl("msa_lm_head_greedy_select_f16", x, Ep, logits, workspace, M, V, K,
                             temperature, banned_host, n_banned, stop_host, n_stop, finished,
                             row_mode, force_eos_all, eos_idx, tok, tok_stride, score,
                             score_stride, len_dev, stream);
}

// ---- the entry point that allocates nothing ---------------------------------------------------
// The per-row, per-workgroup selection partials of the fused vocabulary projection live in a
// fixed device array instead of a caller-provided workspace, for callers that cannot allocate
// device memory (code under graph capture, serving loops, harnesses that forbid it).  Every
// GPU the library runs on holds its own copy of the array (512 KiB) until the process ends.
// In host code the array's name is only a stand-in for the symbol: the address the kernels get
// is looked up once per device with hipGetSymbolAddress and kept in g_scratch_ptr.
constexpr int NA_MAX_ROWS = 64;    // activation rows
constexpr int NA_MAX_PARTS = 256;  // workgroups of the projection = partials per row
static __device__ __align__(256) unsigned char
    scratch[NA_MAX_ROWS * NA_MAX_PARTS * sizeof(SelectPartial)];

namespace {
constexpr int NA_MAX_DEVICES = 64;
std::mutex g_scratch_mutex;
void* g_scratch_ptr[NA_MAX_DEVICES] = {};

// the current device's copy of `scratch`; NULL (with the error text set) on failure
void* scratch_for_current_device(const char* name) {
  int dev = -1;
  hipError_t e = hipGetDevice(&dev);
  if (e != hipSuccess || dev < 0 || dev >= NA_MAX_DEVICES) {
    msa_set_error("%s: no usable current device (%s, device %d)", name, hipGetErrorString(e), dev);
    return nullptr;
  }
  std::lock_guard<std::mutex> lock(g_scratch_mutex);
  if (!g_scratch_ptr[dev]) {
    void* p = nullptr;
    e = hipGetSymbolAddress(&p, HIP_SYMBOL(scratch));
    if (e != hipSuccess || !p) {
      msa_set_error("%s: hipGetSymbolAddress(scratch) failed on device %d: %s", name, dev,
                    hipGetErrorString(e));
      return nullptr;
    }
    g_scratch_ptr[dev] = p;
  }
  return g_scratch_ptr[dev];
}
}  // namespace

extern "C" int msa_lm_head_greedy_select_noalloc_f16(
    const void* x, const void* Ep, void* logits, int M, int V, int K, float temperature,
    const int32_t* banned_host, int n_banned, const int32_t* stop_host, int n_stop,
    uint8_t* finished, const uint8_t* row_mode, int force_eos_all, int eos_idx, int64_t* tok,
    int64_t tok_stride, float* score, int64_t score_stride, const int32_t* len_dev, void* stream) {
  const char* name = "msa_lm_head_greedy_select_noalloc_f16";
  MSA_REQUIRE(M >= 1 && M <= NA_MAX_ROWS, MSA_ERR_CAPACITY,
              "%s: M=%d rows exceed the %d the fixed scratch array holds", name, M, NA_MAX_ROWS);
  MSA_REQUIRE(num_cus() <= NA_MAX_PARTS, MSA_ERR_CAPACITY,
              "%s: %d compute units exceed the %d partials per row the fixed scratch array holds",
              name, num_cus(), NA_MAX_PARTS);
  void* ws = scratch_for_current_device(name);
  if (!ws) return MSA_ERR_HIP;
  // every partial the combine kernel reads is written by the projection of the same call, so
  // nothing in the array has to start at zero
  return lm_head_select_impl(name, x, Ep, logits, ws, M, V, K, temperature, banned_host, n_banned,
                             stop_host, n_stop, finished, row_mode, force_eos_all, eos_idx, tok,
                             tok_stride, score, score_stride, len_dev, stream);
}

extern "C" int msa_linear_default_splits(int64_t M, int N, int K) {
  return pick_splits(M, N, K, 2);
}

extern "C" int msa_linear_default_splits_w8a16(int64_t M, int N, int K) {
  return pick_splits(M, N, K, 1);
}

extern "C" int msa_linear_default_splits_rows(int64_t M, int N, int K) {
  return pick_row_splits(M, N, K);
}

extern "C" int msa_linear_f16(const void* x, const void* Wp, const void* bias,
                              const void* residual, void* y, int64_t M, int N, int K,
                              unsigned flags, void* stream) {
  return linear_entry<false>("msa_linear_f16", x, Wp, nullptr, bias, residual, y, M, N, K, flags,
                             stream);
}

extern "C" int msa_linear_w8a16(const void* x, const int8_t* Wq, const void* scales,
                                const void* bias, const void* residual, void* y, int64_t M, int N,
                                int K, unsigned flags, void* stream) {
  return linear_entry<true>("msa_linear_w8a16", x, Wq, scales, bias, residual, y, M, N, K, flags,
                            stream);
}

extern "C" int msa_linear_partial_f16(const void* x, const void* Wp, float* part, int64_t M, int N,
                                      int K, int S, unsigned flags, void* stream) {
  return partial_entry<false>("msa_linear_partial_f16", x, Wp, nullptr, part, M, N, K, S, flags,
                              stream);
}

extern "C" int msa_linear_partial_w8a16(const void* x, const int8_t* Wq, const void* scales,
                                        float* part, int64_t M, int N, int K, int S,
                                        unsigned flags, void* stream) {
  return partial_entry<true>("msa_linear_partial_w8a16", x, Wq, scales, part, M, N, K, S, flags,
                             stream);
}

extern "C" int msa_qkv_proj_f16(const void* x, const void* Wqkv, const void* bqkv, void* q_out,
                                void* Kcache, void* Vcache, int B, int T, int H, int hd, int S0,
                                int S_cap, int K, unsigned flags, const int32_t* len_dev,
                                void* stream) {
  return qkv_entry<false>("msa_qkv_proj_f16", x, Wqkv, nullptr, bqkv, q_out, Kcache, Vcache, B, T,
                          H, hd, S0, S_cap, K, flags, len_dev, stream);
}

extern "C" int msa_qkv_proj_w8a16(const void* x, const int8_t* Wq, const void* scales,
                                  const void* bqkv, void* q_out, void* Kcache, void* Vcache, int B,
                                  int T, int H, int hd, int S0, int S_cap, int K, unsigned flags,
                                  const int32_t* len_dev, void* stream) {
  return qkv_entry<true>("msa_qkv_proj_w8a16", x, Wq, scales, bqkv, q_out, Kcache, Vcache, B, T, H,
                         hd, S0, S_cap, K, flags, len_dev, stream);
}
