/*
 * metaseq_hybrid.h - C ABI of libmetaseq_hybrid.so: gfx950 kernels and the step function of hybrid
 * decoders, i.e. models whose layers mix attention (over a cached latent, or grouped within chunks)
 * with recurrent layers (gated linear recurrent units, gated delta rule), one after the other or side
 * by side, and dense or routed feed-forwards.
 *
 * Conventions are those of metaseq_amd.h (device pointers, a hipStream_t as `stream`, 0 or a negative
 * msa_status, nothing allocates or synchronises).  In addition:
 *
 *   - Formats.  `dtype` MSA_BF16: activations and the cached latent are bf16, matrices are bf16
 *     in the tile-packed layout of metaseq_amd.h (16 x 32 blocks in MFMA lane order).  MSA_F32:
 *     everything is fp32, matrices row-major.  In both, the residual stream, norms, routing,
 *     recurrent state, attention scores and softmax are fp32, and so are all vectors (norm weights,
 *     biases, convolution taps, decay parameters).
 *   - Padding.  Every matrix dimension is padded with zeros by the caller to what the kernels want
 *     (below); an element count that enters a mean is passed separately.  A reduction length K is
 *     a multiple of 64 and at least 128 for linear layers, a multiple of 32 for grouped ones.
 *   - Batches are flat: M tokens in nseg contiguous segments, each the next tokens of one cache slot.
 *     Prefill, a portion of a prompt, a decode step and any mix of them are the same call.
 */
#ifndef METASEQ_HYBRID_H
#define METASEQ_HYBRID_H

#include "metaseq_amd.h"

#ifdef __cplusplus
extern "C" {
#endif

enum { MSA_BF16 = 0, MSA_F32 = 1 };
enum { MSA_GLU_NONE = -1, MSA_GLU_GELU = 0, MSA_GLU_CLAMPED = 1 };
enum { MSA_ACT_NONE = 0, MSA_ACT_RELU2 = 1 };
enum { MSA_GATE_SILU = 0, MSA_GATE_SIGMOID = 1 };
enum { MSA_MIX_LATENT = 0, MSA_MIX_RGLRU = 1, MSA_MIX_DELTA = 2, MSA_MIX_PARALLEL = 3 };
enum { MSA_FF_NONE = 0, MSA_FF_DENSE = 1, MSA_FF_MOE = 2, MSA_FF_RELU2 = 3 };
#define MSA_OUT2_PACKED 16u /* msa_linear: y2 in the packed layout */

/* A flat batch.  tok_*: per token its cache slot, its position in the slot's sequence (negative: the
 * token is inactive - it changes no cache or state, its outputs mean nothing) and its offset in its
 * segment.  seg_*: first token of every segment (nseg + 1 entries), slot, position of its first
 * token (negative: inactive).  host_*: host copies of seg_start / seg_slot / seg_pos, needed
 * unless every segment holds one token.  key_bound: no token sees more than this many keys. */
typedef struct {
  int M, nseg, max_count, key_bound;
  const int32_t *tok_slot, *tok_pos, *tok_off;
  const int32_t *seg_start, *seg_slot, *seg_pos;
  const int32_t *host_start, *host_slot, *host_pos;
} msa_batch;

/* y[m, n] = sum_k x[m, k] W[n, k].  Columns n < n32 are stored in the activation format, row-major
 * with stride n32 (or packed, MSA_OUT_PACKED), the columns from n32 on as fp32 into y32[M, N - n32].
 * glu: the columns below n32 are (gate, up) pairs 2i, 2i + 1 and column i of y receives the gated
 * activation (MSA_GLU_GELU: gelu_tanh(g) u; MSA_GLU_CLAMPED: with g' = min(g, limit) and
 * u' = clamp(u, +-limit), g' sigmoid(1.702 g') (u' + 1)); y then has stride n32 / 2.
 * N and n32 are multiples of 16 (n32 of 32 with glu).  bf16: M <= 128 rows may be packed. */
int msa_linear_bf16(const void* x, const void* W, void* y, float* y32, int64_t M, int N, int K,
                    int n32, int glu, float limit, unsigned flags, void* stream);
int msa_linear_f32(const float* x, const float* W, float* y, float* y32, int64_t M, int N, int K,
                   int n32, int glu, float limit, void* stream);
/* fp32 sums of S slices of K, part[S][M][N]; msa_linear_bf16_splits picks S (packed: M <= 128). */
int msa_linear_partial_bf16(const void* x, const void* W, float* part, int64_t M, int N, int K, int S,
                            unsigned flags, void* stream);
int msa_linear_bf16_splits(int64_t M, int N, int K, int packed);

/* A linear layer with what follows it: z = x W^T + bias ; columns below n32 leave as act(z) in the
 * activation format, those of them from n2 on into a matrix of their own (y2 [M, n32 - n2]; y2 NULL: all
 * into y, otherwise y is [M, n2]) ; the columns from n32 on leave as fp32 into y32 [M, N - n32], with
 * decay_rate as decays exp(-decay_rate[n - n32] softplus(z)).  MSA_ACT_RELU2: max(z, 0)^2.  bias [N] and
 * decay_rate [N - n32] may be NULL.  n2 and n32 are multiples of 16.  flags (bf16): MSA_IN_PACKED,
 * MSA_OUT_PACKED (y), MSA_OUT2_PACKED (y2). */
typedef struct {
  int dtype;
  const void *x, *W;
  int64_t M;
  int N, K, n32, n2, act;
  unsigned flags;
  const float *bias, *decay_rate;
  void *y, *y2;
  float* y32;
} msa_linear_args;
int msa_linear(const msa_linear_args* a, void* stream);

/* Grouped products: group g multiplies its own columns of x, or its own rows, by its own matrix.
 * Dense (tile_group NULL): y[m, g * y_group + n] = sum_k x[m, g * x_group + k] W_g[n, k] for all M rows
 * and `groups` groups.  Routed: the tiles of a msa_moe_plan; row r of group g's sorted rows reads x row
 * perm[r] / rows_per_x (perm NULL: x row r) and writes y row r.  x_mb / y_mb > 0: packed layout with
 * that many row blocks (bf16 only).  y_f32: fp32 output.  glu as above (y has N / 2 columns).
 * Routed tiles have 16, 32 or 64 rows, or 256 (bf16 row-major, K % 64 == 0, K >= 128).
 * x_groups > 0: group g reads column group g % x_groups.  y_row0 is added to every row of y. */
typedef struct {
  int dtype;
  const void* x; int64_t ldx; int x_group, x_groups, x_mb;
  const void* W;
  void* y; int64_t ldy; int y_group, y_mb, y_f32, y_row0;
  int N, K, groups, glu;
  float limit;
  int64_t M;
  const int32_t *perm, *tile_group, *tile_row, *n_tiles, *group_end;
  int rows_per_x, max_tiles, tile_rows;
} msa_group_linear_args;
int msa_group_linear(const msa_group_linear_args* a, void* stream);

/* Routing of M tokens over E experts: softmax over the logits z (row stride ldz), the experts of the
 * `keep` groups (of n_groups equal ones) with the largest maximum are eligible, the `top` largest
 * are chosen; ids / weights [M, top] (weight = softmax value * scale).  shared_gate (or NULL):
 * sigmoid(z[m, E]). */
int msa_moe_route(const float* z, int ldz, int M, int E, int n_groups, int keep, int top, float scale,
                  int32_t* ids, float* weights, float* shared_gate, void* stream);
/* Sorts the P = M * top (token, choice) pairs by expert: perm[r] = pair at sorted row r, inverse[pair] =
 * r, group_end[E] = end of every expert's rows, and the list of tiles of at most tile_rows rows
 * (tile_group, tile_row: first row; n_tiles).  max_tiles entries are provided:
 * P / tile_rows + min(E, P) suffice. */
int msa_moe_plan(const int32_t* ids, int P, int E, int tile_rows, int32_t* perm, int32_t* inverse,
                 int32_t* group_end, int32_t* tile_group, int32_t* tile_row, int32_t* n_tiles,
                 int max_tiles, void* stream);

/* e = table[token] * scale + sinusoid(pos), x = e + step, h = rmsnorm(x) * w (activation format).
 * table: bf16 [vocab, Dp]; inv_freq: double [(D + 1) / 2], the angle per position of column pair i (NULL:
 * no sinusoid); step: [Dp] or NULL; e: fp32 [M, Dp], written unless NULL. */
int msa_embed_rmsnorm(int dtype, const int64_t* tokens, const int32_t* tok_pos, int M,
                      const void* table, int vocab, float scale, const double* inv_freq, int D, int Dp,
                      float eps, const float* step, float* e, float* x, const float* w, void* h, int h_mb,
                      void* stream);
/* The tail of a sublayer: b = sum of S slices part[S][M][Dp] (times gate[m]) + bias + sum_k pair_w[m, k]
 * * pair_y[inverse[m, k]] ; x += rmsnorm(b) * w_post (w_post NULL: x += b) ; with part2 (S2 slices) also
 * x += rmsnorm(part2) * w_post2 ; x is written to probe ; x += add + step (what comes between two layers)
 * ; h = rmsnorm(x) * w_next (w_next NULL: no h).  part or pair_y may be NULL, and bias [Dp], part2, probe
 * [M, Dp], add [M, Dp] and step [Dp]. */
typedef struct {
  int dtype, M, D, Dp, S, S2, top, h_mb;
  float eps;
  const float *part, *gate, *pair_w;
  const void* pair_y;
  const int32_t* inverse;
  const float *bias, *part2, *w_post2, *add, *step;
  float* probe;
  const float *w_post, *w_next;
  float* x;
  void* h;
} msa_tail_args;
int msa_residual_rmsnorm_tail(const msa_tail_args* a, void* stream);

/* Causal convolution per channel over each segment, out = act(conv(in + in_bias) + bias) with act =
 * silu or none; `in` row-major with stride ld_in, C channels, weight [taps, C] (last row: the
 * current token).  state[slot][taps - 1][C]: the last inputs (without in_bias), read here; written by
 * msa_conv_state, or here where every segment holds one token. */
int msa_short_conv(int dtype, const void* in, int64_t ld_in, int C, int taps, const float* in_bias,
                   const float* weight, const float* bias, int silu, void* out, int64_t ld_out,
                   void* state, const msa_batch* b, void* stream);
int msa_conv_state(int dtype, const void* in, int64_t ld_in, int C, int taps, void* state,
                   const msa_batch* b, void* stream);

/* Gated linear recurrent unit over C channels: r, i = sigmoid(gates + gate_bias) (gates: fp32
 * [M, 2C], r then i; overwritten), log a = -8 r softplus(lam), S = a S + sqrt(1 - a^2) i u,
 * out = S gelu_tanh(y + y_bias), packed with out_mb row blocks or row-major (ld_out).
 * carry: fp32 [nseg][chunks][2][C], chunks = msa_rglru_chunks(max_count). */
int msa_rglru_chunks(int max_count);
int msa_rglru_scan(int dtype, float* gates, const float* gate_bias, const float* lam, const void* u,
                   int64_t ld_u, const void* y, int64_t ld_y, const float* y_bias, int C,
                   float* state, float* carry, void* out, int64_t ld_out, int out_mb,
                   const msa_batch* b, void* stream);

/* Gated delta rule.  Per head: S <- g S ; u = beta (v - S^T k) ; S <- S + k u^T ; o = S^T q.  qkv:
 * activations after the convolution, [q: kv_heads x dp | k | v: heads x vp] with stride ld.  ba: fp32
 * [M, ldba], beta logits, then decay logits, per head.  With decay (fp32 [M, heads * dp], the decays
 * themselves) every key channel decays by itself, ba holds beta logits only, and decay_rate and dt_bias are
 * unused.  State fp32 [slot][head][vp][dp]; o: fp32 [M, heads * vp].  dp is 32, 64, 96, 128, 192 or 256,
 * vp a multiple of 16; dim is the unpadded key size. */
typedef struct {
  int dtype, heads, kv_heads, dim, dp, vdim, vp, gate_act;
  const void* qkv; int64_t ld;
  const float* ba; int ldba;
  const float *decay_rate, *dt_bias, *decay;
  float* state;
  float* o;               /* msa_delta_scan writes, msa_delta_output reads */
  const void* gate; int64_t ld_gate;   /* heads * vp columns, activation format */
  const float* w; float eps;           /* the output's norm over vdim, weight [vp] */
  void* out; int64_t ld_out; int out_mb;
} msa_delta_args;
int msa_delta_scan(const msa_delta_args* a, const msa_batch* b, void* stream);
/* out = rmsnorm over vdim of every head's o, times w, times silu(gate) or sigmoid(gate) (gate_act) */
int msa_delta_output(const msa_delta_args* a, int M, void* stream);
/* Both in one launch where every segment holds one token. */
int msa_delta_step(const msa_delta_args* a, const msa_batch* b, void* stream);

/* Attention of several query heads per key/value head over cached keys and values, causal, and within
 * chunks of `chunk` positions (0: one chunk): position i sees j <= i of its own chunk.  q, k, v: columns of
 * the step's rows, all with stride ld (q [M, heads * hd], k [M, kv_heads * hd], v [M, kv_heads * vd]).  A
 * slot's cache holds `rows` positions, k_cache [slot][kv_heads][rows][hd] and v_cache [slot][kv_heads][rows]
 * [vd], the position at its distance from the chunk's start: rows is at least min(capacity, chunk).  Keys
 * of the step's own tokens are read from the step's rows, so what a segment appends may take the place
 * of an older chunk.  gate: fp32 logits [M, ld_gate] per head or NULL: the output is multiplied by their
 * sigmoid.  out: activation format, heads * vd columns.  Rotary: dimension i < rot_dims / 2 of a head is
 * rotated with i + rot_dims / 2 by position * inv_freq[i] (double, device). */
typedef struct {
  int dtype, heads, kv_heads, hd, vd, chunk, rot_dims, rows;
  float scale;
  const double* inv_freq;
  void *q, *k, *v; int64_t ld;
  void *k_cache, *v_cache;
  const float* gate; int ld_gate;
  void* out; int64_t ldo; int out_mb;
  float* partial;         /* splits > 1: [M][heads][splits][vd + 4] */
  int splits;
  int fused;              /* the attention kernel rotates and appends (msa_grouped_fuses) */
} msa_grouped_args;
/* rotates q and k in place; where every segment holds one token, also appends keys and values */
int msa_grouped_rotate(const msa_grouped_args* a, const msa_batch* b, void* stream);
/* appends the keys and values of every segment's last chunk (nothing where msa_grouped_rotate did) */
int msa_grouped_append(const msa_grouped_args* a, const msa_batch* b, void* stream);
int msa_grouped_attention_splits(const msa_grouped_args* a, int M, int key_bound);
/* whether msa_grouped_attention can take rotation and appending over for this batch: with `fused` set, the
 * other two calls fall away */
int msa_grouped_fuses(const msa_grouped_args* a, const msa_batch* b);
/* The outputs of segments seg0 .. seg1 - 1: all of them of one token each (longest == 1), or of any size up
 * to `longest`, after msa_grouped_rotate and before msa_grouped_append (unless fused).  Head sizes: fp32, and bf16 beyond
 * 256, up to 1024; bf16 64, 128, 192 or 256. */
int msa_grouped_attention(const msa_grouped_args* a, const msa_batch* b, int seg0, int seg1, int longest,
                          void* stream);

/* Latents: part = fp32 sums [S][M][N] of the down-projections, columns [0, qp) the query latent,
 * [qp, qp + rp) the key/value latent (absent with latent NULL).  Both RMS-normed over their q_rank /
 * kv_rank true elements; cq in activation format, the key/value latent into
 * latent[slot][capacity][rp] at the token's position. */
int msa_latent_norm(int dtype, const float* part, int S, int N, int M, int q_rank, int qp,
                    const float* wq, int kv_rank, int rp, const float* wkv, float eps, void* cq,
                    int cq_mb, void* latent, int capacity, const msa_batch* b, void* stream);
/* Causal softmax attention in the latent space: q [M, heads, rp] (already multiplied by the key
 * up-projection), keys = values = the slot's latents; out [M, heads, rp] in activation format.
 * splits > 1: partial [M][heads][splits][rp + 4] fp32. */
int msa_latent_attention_splits(int dtype, int M, int heads, int rp, int key_bound);
int msa_latent_attention(int dtype, const void* q, const void* latent, int capacity, int heads, int rp,
                         float scale, void* out, float* partial, int splits,
                         const int32_t* tok_slot, const int32_t* tok_pos, int M, void* stream);
/* Causal attention of T new queries at positions pos0 .. over S = pos0 + T expanded keys and values
 * (bf16): q [T, ldq] (head h at h * hd), kv [S, ldkv] (key of head h at h * hd, its value at
 * (heads + h) * hd); rows row0 .. of out, row-major (ldo) or packed with out_mb row blocks.
 * hd: 32, 64, 96, 128, 192 or 256. */
int msa_flash_attention_bf16(const void* q, int64_t ldq, const void* kv, int64_t ldkv, void* out,
                             int64_t ldo, int out_mb, int row0, int heads, int hd, int T, int pos0,
                             float scale, void* stream);

/* clears columns c0 .. c1 - 1 of an activation matrix */
int msa_zero_columns(int dtype, void* y, int64_t M, int64_t ld, int mb, int c0, int c1, void* stream);
/* rows `rows[i]` of an activation matrix (layout src_mb / ld) to row i of another (dst_mb) */
int msa_gather_rows(int dtype, const void* src, int src_mb, const int32_t* rows, int n, int K, void* dst,
                    int dst_mb, void* stream);
/* step_pos[b] = lens[b] if row b is active (lens >= 0) and tokens[b] != pad, else -1 */
int msa_step_positions(const int32_t* lens, const int64_t* tokens, int64_t tok_stride, int64_t pad,
                       int B, int32_t* step_pos, void* stream);
/* lens[b] += 1 where step_pos[b] >= 0 */
int msa_advance_active(int32_t* lens, const int32_t* step_pos, int B, void* stream);

/* ---- the step function ----------------------------------------------------------------------- */
/* the attention side of a parallel mixer */
typedef struct {
  int heads, kv_heads, hd, vd, chunk, rot_dims, ko;
  float scale;
  const double* inv_freq; /* device, [rot_dims / 2] */
  const void* w_out;      /* [Dp, ko]; NULL where both sides' ko are equal: the layer's w_out is
                             [Dp, 2 ko], this side's columns behind the delta rule's */
  const float* out_norm;  /* [Dp] */
} msa_attention_layer;

typedef struct {
  int kind; /* MSA_MIX_* */
  /* latent attention */
  int heads, hd, q_rank, qp, kv_rank, rp, kv_from; /* kv_from: layer that owns the latent, or -1 */
  float scale;
  const void *w_in;     /* [qp (+ rp), Dp]: down-projections                                        */
  const void *w_q;      /* [heads * hd, qp]                                                         */
  const void *w_kv;     /* [2 * heads * hd, rp]: key rows, then value rows (bf16 only)               */
  const void *w_absorb; /* per head [rp, hd]: transposed key up-projection                           */
  const void *w_v;      /* per head [hd, rp]                                                         */
  const float *wq_norm, *wkv_norm;
  /* recurrent layers: heads, kv_heads, dim, dp, vdim, vp (delta); channels, blocks (rglru)            */
  int kv_heads, dim, dp, vdim, vp, channels, blocks, taps;
  const float *conv_w, *conv_b, *in_bias, *y_bias, *gate_bias, *lam, *decay_rate, *dt_bias, *o_norm;
  const void* w_gates;  /* per block r, then per block i: [2 * blocks][channels / blocks]^2          */
  /* parallel: grouped attention (att) beside a delta rule with channel decays, the sum of their normed
   * outputs (out_norm: the delta side's).  w_in's columns, with in_bias per column: attention's q, k, v ;
   * the delta rule's q, k, v ; lr columns of low-rank inputs ; fp32 from there on: a gate logit per
   * attention head, a beta logit per delta head.  w_lr [heads * (vp + dp), lr]: the read-out gate's columns,
   * then the decays' (lr_bias per column, lr_rate [heads * dp]). */
  msa_attention_layer att;
  int lr;
  const void* w_lr;
  const float *lr_bias, *lr_rate, *out_norm;
  /* all */
  const void* w_out;    /* [Dp, ko]                                                                 */
  int n_in, ko;
  const float *norm1, *norm1b, *norm2, *norm2b; /* norm1b, norm2b: after the sublayer, or NULL */
  /* feed-forward */
  int ff_kind, ff, experts, top, n_groups, keep, ff_expert, ff_shared; /* padded sizes */
  float router_scale, limit_expert, limit_shared;
  const void* w_ff_in;  /* dense: (gate, up) row pairs [2 ff, Dp]; relu2: [ff, Dp]; moe: shared expert's pairs, then
                           router rows and the shared gate's row as fp32 columns                     */
  int n_ff_in;
  const float *ff_bias, *ff_down_bias; /* relu2: [ff], [Dp] */
  const void* w_ff_down; /* dense, relu2 or shared expert (NULL: none) */
  const void *w_e_in, *w_e_down; /* per expert [2 ff_expert, Dp] pairs, [Dp, ff_expert] */
} msa_hybrid_layer;

typedef struct {
  int dtype, layers, D, Dp, vocab, Vp;
  float eps, embed_scale;
  const void* embed;      /* bf16 [vocab, Dp] */
  const double* inv_freq; /* device; NULL: no positions are added to the embedding */
  const float* final_norm;
  const void* head;       /* [Vp, Dp] */
  /* The layers in the order they run (host arrays, copied; n_runs 0: once each).  A run whose run_pass is
   * t >= 0 begins pass t of a loop: loop_step[t] is added to the residual stream in front of it, and, for
   * t > 0, the embedding.  Every run has its own cache and state. */
  int n_runs;
  const int32_t *run_layer, *run_pass;
  const float* loop_step; /* device, [passes][Dp] */
} msa_hybrid_config;

typedef struct msa_hybrid msa_hybrid;
int msa_hybrid_create(const msa_hybrid_config* cfg, const msa_hybrid_layer* layers, msa_hybrid** out);
void msa_hybrid_destroy(msa_hybrid* d);

/* Cache pointers per run of a layer: latent [slots][capacity][rp] (attention layers that own one), conv
 * [slots][taps - 1][channels] and rec (rglru: [slots][channels], delta: [slots][heads][vp][dp]), keys and
 * values [slots][kv_heads][kv_rows][hd or vd]. */
typedef struct {
  void *latent, *conv;
  float* rec;
  void *keys, *values;
  int kv_rows;
} msa_hybrid_state;

typedef struct {
  msa_batch batch;
  const int64_t* tokens;   /* [M] */
  const msa_hybrid_state* state; /* host array, one per run */
  int capacity;            /* positions per slot */
  const int32_t* rows;     /* device: rows whose logits are wanted, or NULL = all */
  int n_rows;
  float* logits;           /* [n_rows or M][Vp]; NULL: none */
  float* probe;            /* [runs][M][Dp]: the residual stream after every run of a layer, or NULL */
  void* workspace;
  int64_t workspace_bytes;
} msa_hybrid_step_args;
int64_t msa_hybrid_workspace_bytes(const msa_hybrid* d, const msa_hybrid_step_args* a);
int msa_hybrid_step(const msa_hybrid* d, const msa_hybrid_step_args* a, void* stream);

#ifdef __cplusplus
}
#endif
#endif
