// The step function of a hybrid decoder: one call runs a flat batch (prompts, portions of prompts,
// decode steps, any mix) through embedding, layers and vocabulary projection, launching the
// kernels back to back on the caller's stream from a table of device pointers.
//
// Up to 128 tokens the matrix products run on the weight-streaming kernels with packed activations
// (split-K sums finished by the norm tail), beyond on the MFMA tile kernels with row-major ones.
// Latent attention: segments of more than EXPAND_FROM new tokens expand keys and values per head, shorter
// ones attend in the latent space.
#include <stdlib.h>
#include <string.h>

#include <new>

#include "common.h"

namespace {

// one run of a layer (a layer of a loop runs several times)
struct LayerRun {
  int layer;
  int pass;   // >= 0: this run begins that pass of a loop
  int owner;  // run whose latent it attends to (latent attention)
};

}  // namespace

struct msa_hybrid {
  msa_hybrid_config cfg;
  msa_hybrid_layer* layers;
  LayerRun* runs;
  bool adds_embedding;  // some pass of a loop begins with the embedding
};

namespace {

constexpr int EXPAND_FROM = 16;

#define HY(call)              \
  do {                        \
    const int rc_ = (call);   \
    if (rc_) return rc_;      \
  } while (0)

// An activation matrix of n columns in the step's format; ld > n: some columns of a wider one.
struct Act {
  void* p;
  int ld, n;
};

struct Run {
  const msa_hybrid* d;
  const msa_hybrid_step_args* a;
  void* stream;
  bool dry;  // only measure the workspace
  bool f32;
  int M, mb, es;  // rows, row blocks of packed activations (0: row-major), bytes per element
  char* base;
  int64_t off, peak;

  void* alloc(int64_t bytes) {
    void* p = base + off;
    off += (bytes + 255) & ~(int64_t)255;
    if (off > peak) peak = off;
    return p;
  }
  Act act(int ld) { return {alloc((int64_t)(mb > 0 ? mb * 16 : M) * ld * es), ld, ld}; }
  // n columns of x from c on (a multiple of 32)
  Act columns(const Act& x, int c, int n) const {
    return {(char*)x.p + (int64_t)c * (mb > 0 ? mb * 16 : 1) * es, x.ld, n};
  }
  unsigned in_flags() const { return mb > 0 ? MSA_IN_PACKED : 0u; }

  // y (row-major or, with glu, in the activation layout) = x W^T with fp32 tail columns
  int linear(const Act& x, const void* W, void* y, bool y_act, float* y32, int N, int n32, int glu,
             float limit) {
    if (dry) return MSA_OK;
    if (f32)
      return msa_linear_f32((const float*)x.p, (const float*)W, (float*)y, y32, M, N, x.ld, n32, glu,
                            limit, stream);
    return msa_linear_bf16(x.p, W, y, y32, M, N, x.ld, n32, glu, limit,
                           in_flags() | (y_act && mb > 0 ? MSA_OUT_PACKED : 0u), stream);
  }
  // fp32 sums of S slices
  float* partial(const Act& x, const void* W, int N, int& S, int& rc, int least = 1) {
    S = f32 ? 1 : msa_linear_bf16_splits(M, N, x.ld, mb > 0);
    if (least > 1) {  // slices that do not cross the borders of `least` equal parts of K
      S = S > least ? S : least;
      while (S > least && x.ld % (64 * S)) S /= 2;
    }
    float* part = (float*)alloc((int64_t)S * M * N * 4);
    rc = MSA_OK;
    if (dry) return part;
    if (f32)
      rc = msa_linear_f32((const float*)x.p, (const float*)W, nullptr, part, M, N, x.ld, 0, MSA_GLU_NONE,
                          0.f, stream);
    else
      rc = msa_linear_partial_bf16(x.p, W, part, M, N, x.ld, S, in_flags(), stream);
    return part;
  }
  int zero_tail(const Act& y, int used) {
    if (dry || used == y.n) return MSA_OK;
    return msa_zero_columns(d->cfg.dtype, y.p, M, y.ld, mb, used, y.n, stream);
  }

  // y, y2 (activation format; y row-major), y32 = a linear layer with bias, activation, decays
  int linear_post(const Act& x, const void* W, int N, int n32, const float* bias, int act,
                  const float* rate, void* y, bool y_act, const Act* y2, float* y32) {
    if (dry) return MSA_OK;
    msa_linear_args l{};
    l.dtype = d->cfg.dtype;
    l.x = x.p;
    l.W = W;
    l.M = M;
    l.N = N;
    l.K = x.ld;
    l.n32 = n32;
    l.bias = bias;
    l.act = act;
    l.decay_rate = rate;
    l.y = y;
    l.y32 = y32;
    l.flags = in_flags() | (y_act && mb > 0 ? MSA_OUT_PACKED : 0u);
    if (y2) {
      l.y2 = y2->p;
      l.n2 = n32 - y2->ld;
      if (mb > 0) l.flags |= MSA_OUT2_PACKED;
    }
    return msa_linear(&l, stream);
  }

  int latent(int ri, const Act& h, Act& out);
  int latent_rows(const msa_hybrid_layer& l, void* cache, void* q, Act& out, int r0, int r1);
  int latent_segment(const msa_hybrid_layer& l, void* cache, void* q, Act& out, int seg);
  int rglru(int ri, const Act& h, Act& out);
  int delta(int ri, const Act& h, Act& out);
  int delta_core(const msa_hybrid_layer& l, const msa_hybrid_state& st, char* in, int64_t ld,
                 msa_delta_args& t, Act& out);
  int grouped(const msa_hybrid_layer& l, const msa_hybrid_state& st, char* in, int64_t ld,
              const float* gate, int ld_gate, Act& out);
  int parallel(int ri, const Act& h, Act& left, Act& right);
  int feed_forward(const msa_hybrid_layer& l, msa_tail_args& t);
  int tail(const msa_tail_args& t) { return dry ? MSA_OK : msa_residual_rmsnorm_tail(&t, stream); }
  int go();
};

int Run::latent_rows(const msa_hybrid_layer& l, void* cache, void* q, Act& out, int r0, int r1) {
  const int n = r1 - r0;
  const int64_t save = off;
  void* qa = alloc((int64_t)n * l.heads * l.rp * es);
  void* ol = alloc((int64_t)n * l.heads * l.rp * es);
  const int splits =
      msa_latent_attention_splits(d->cfg.dtype, n, l.heads, l.rp, a->batch.key_bound);
  float* part = splits > 1 ? (float*)alloc((int64_t)n * l.heads * splits * (l.rp + 4) * 4) : nullptr;
  if (!dry) {
    msa_group_linear_args g{};
    g.dtype = d->cfg.dtype;
    g.glu = MSA_GLU_NONE;
    g.groups = l.heads;
    g.M = n;
    g.x = (char*)q + (int64_t)r0 * l.heads * l.hd * es;
    g.ldx = (int64_t)l.heads * l.hd;
    g.x_group = l.hd;
    g.W = l.w_absorb;
    g.y = qa;
    g.ldy = (int64_t)l.heads * l.rp;
    g.y_group = l.rp;
    g.N = l.rp;
    g.K = l.hd;
    HY(msa_group_linear(&g, stream));
    HY(msa_latent_attention(d->cfg.dtype, qa, cache, a->capacity, l.heads, l.rp, l.scale, ol, part,
                            splits, a->batch.tok_slot + r0, a->batch.tok_pos + r0, n, stream));
    g.x = ol;
    g.ldx = (int64_t)l.heads * l.rp;
    g.x_group = l.rp;
    g.W = l.w_v;
    g.y = out.p;
    g.ldy = out.ld;
    g.y_group = l.hd;
    g.y_mb = mb;
    g.y_row0 = r0;
    g.N = l.hd;
    g.K = l.rp;
    HY(msa_group_linear(&g, stream));
  }
  off = save;
  return MSA_OK;
}

int Run::latent_segment(const msa_hybrid_layer& l, void* cache, void* q, Act& out, int seg) {
  const msa_batch& b = a->batch;
  const int r0 = b.host_start[seg], n = b.host_start[seg + 1] - r0, pos0 = b.host_pos[seg];
  const int S = pos0 + n, width = 2 * l.heads * l.hd;
  const int64_t save = off;
  void* kv = alloc((int64_t)S * width * es);
  if (!dry) {
    const char* rows = (char*)cache + (int64_t)b.host_slot[seg] * a->capacity * l.rp * es;
    HY(msa_linear_bf16(rows, l.w_kv, kv, nullptr, S, width, l.rp, width, MSA_GLU_NONE, 0.f, 0, stream));
    HY(msa_flash_attention_bf16((char*)q + (int64_t)r0 * l.heads * l.hd * es, (int64_t)l.heads * l.hd,
                                kv, width, out.p, out.ld, mb, r0, l.heads, l.hd, n, pos0, l.scale,
                                stream));
  }
  off = save;
  return MSA_OK;
}

int Run::latent(int ri, const Act& h, Act& out) {
  const msa_hybrid_layer& l = d->layers[d->runs[ri].layer];
  const msa_batch& b = a->batch;
  const bool owner = l.kv_from < 0;
  void* cache = dry ? nullptr : a->state[d->runs[ri].owner].latent;
  int S, rc;
  float* part = partial(h, l.w_in, l.n_in, S, rc);
  HY(rc);
  Act cq = act(l.qp);
  if (!dry)
    HY(msa_latent_norm(d->cfg.dtype, part, S, l.n_in, M, l.q_rank, l.qp, l.wq_norm, l.kv_rank, l.rp,
                       l.wkv_norm, d->cfg.eps, cq.p, mb, owner ? cache : nullptr, a->capacity, &b,
                       stream));
  const int nq = l.heads * l.hd;
  void* q = alloc((int64_t)M * nq * es);
  HY(linear(cq, l.w_q, q, false, nullptr, nq, nq, MSA_GLU_NONE, 0.f));
  // runs of short segments attend in the latent space, long segments over expanded keys
  if (f32 || b.max_count <= EXPAND_FROM) {
    HY(latent_rows(l, cache, q, out, 0, M));
  } else {
    for (int s = 0; s < b.nseg;) {
      const int n = b.host_start[s + 1] - b.host_start[s];
      if (n > EXPAND_FROM && b.host_pos[s] >= 0) {
        HY(latent_segment(l, cache, q, out, s));
        ++s;
        continue;
      }
      int e = s + 1;
      while (e < b.nseg && (b.host_start[e + 1] - b.host_start[e] <= EXPAND_FROM || b.host_pos[e] < 0))
        ++e;
      HY(latent_rows(l, cache, q, out, b.host_start[s], b.host_start[e]));
      s = e;
    }
  }
  return zero_tail(out, nq);
}

int Run::rglru(int ri, const Act& h, Act& out) {
  const msa_hybrid_layer& l = d->layers[d->runs[ri].layer];
  const msa_batch& b = a->batch;
  const int C = l.channels, bs = C / l.blocks, chunks = msa_rglru_chunks(b.max_count);
  char* yx = (char*)alloc((int64_t)M * l.n_in * es);  // y, then the convolution's input
  HY(linear(h, l.w_in, yx, false, nullptr, l.n_in, l.n_in, MSA_GLU_NONE, 0.f));
  void* u = alloc((int64_t)M * C * es);
  float* gates = (float*)alloc((int64_t)M * 2 * C * 4);
  float* carry = (float*)alloc((int64_t)b.nseg * chunks * 2 * C * 4);
  if (!dry) {
    const msa_hybrid_state& st = a->state[ri];
    char* raw = yx + (int64_t)C * es;
    HY(msa_short_conv(d->cfg.dtype, raw, l.n_in, C, l.taps, l.in_bias, l.conv_w, l.conv_b, 0, u, C,
                      st.conv, &b, stream));
    HY(msa_conv_state(d->cfg.dtype, raw, l.n_in, C, l.taps, st.conv, &b, stream));
    msa_group_linear_args g{};
    g.dtype = d->cfg.dtype;
    g.glu = MSA_GLU_NONE;
    g.groups = 2 * l.blocks;
    g.M = M;
    g.x = u;
    g.ldx = C;
    g.x_group = bs;
    g.x_groups = l.blocks;
    g.W = l.w_gates;
    g.y = gates;
    g.ldy = 2 * C;
    g.y_group = bs;
    g.y_f32 = 1;
    g.N = g.K = bs;
    HY(msa_group_linear(&g, stream));
    HY(msa_rglru_scan(d->cfg.dtype, gates, l.gate_bias, l.lam, u, C, yx, l.n_in, l.y_bias, C, st.rec,
                      carry, out.p, out.ld, mb, &b, stream));
  }
  return zero_tail(out, C);
}

// The delta rule behind its projections: `in` holds q, k, v (row-major, stride ld); t comes with the
// gate, the beta logits and the decays.
int Run::delta_core(const msa_hybrid_layer& l, const msa_hybrid_state& st, char* in, int64_t ld,
                    msa_delta_args& t, Act& out) {
  const msa_batch& b = a->batch;
  const int C = 2 * l.kv_heads * l.dp + l.heads * l.vp;
  void* qkv = alloc((int64_t)M * C * es);
  const bool step = b.max_count == 1;
  t.o = step ? nullptr : (float*)alloc((int64_t)M * l.heads * l.vp * 4);
  if (!dry) {
    HY(msa_short_conv(d->cfg.dtype, in, ld, C, l.taps, nullptr, l.conv_w, nullptr, 1, qkv, C, st.conv, &b,
                      stream));
    HY(msa_conv_state(d->cfg.dtype, in, ld, C, l.taps, st.conv, &b, stream));
    t.dtype = d->cfg.dtype;
    t.heads = l.heads;
    t.kv_heads = l.kv_heads;
    t.dim = l.dim;
    t.dp = l.dp;
    t.vdim = l.vdim;
    t.vp = l.vp;
    t.qkv = qkv;
    t.ld = C;
    t.state = st.rec;
    t.w = l.o_norm;
    t.eps = d->cfg.eps;
    t.out = out.p;
    t.ld_out = out.ld;
    t.out_mb = mb;
    if (step) {
      HY(msa_delta_step(&t, &b, stream));
    } else {
      HY(msa_delta_scan(&t, &b, stream));
      HY(msa_delta_output(&t, M, stream));
    }
  }
  return zero_tail(out, l.heads * l.vp);
}

int Run::delta(int ri, const Act& h, Act& out) {
  const msa_hybrid_layer& l = d->layers[d->runs[ri].layer];
  const int C = 2 * l.kv_heads * l.dp + l.heads * l.vp, n32 = C + l.heads * l.vp;
  char* in = (char*)alloc((int64_t)M * n32 * es);  // q, k, v, gate
  float* ba = (float*)alloc((int64_t)M * (l.n_in - n32) * 4);
  HY(linear(h, l.w_in, in, false, ba, l.n_in, n32, MSA_GLU_NONE, 0.f));
  msa_delta_args t{};
  t.ba = ba;
  t.ldba = l.n_in - n32;
  t.decay_rate = l.decay_rate;
  t.dt_bias = l.dt_bias;
  t.gate_act = MSA_GATE_SILU;
  t.gate = in + (int64_t)C * es;
  t.ld_gate = n32;
  return delta_core(l, dry ? msa_hybrid_state{} : a->state[ri], in, n32, t, out);
}

// Grouped attention behind its projections: `in` holds q, k, v.  Runs of segments of one token each and of
// longer segments have kernels of their own.
int Run::grouped(const msa_hybrid_layer& l, const msa_hybrid_state& st, char* in, int64_t ld,
                 const float* gate, int ld_gate, Act& out) {
  const msa_attention_layer& t = l.att;
  const msa_batch& b = a->batch;
  msa_grouped_args g{};
  g.dtype = d->cfg.dtype;
  g.heads = t.heads;
  g.kv_heads = t.kv_heads;
  g.hd = t.hd;
  g.vd = t.vd;
  g.chunk = t.chunk;
  g.rot_dims = t.rot_dims;
  g.rows = st.kv_rows;
  g.scale = t.scale;
  g.inv_freq = t.inv_freq;
  g.q = in;
  g.k = in + (int64_t)t.heads * t.hd * es;
  g.v = (char*)g.k + (int64_t)t.kv_heads * t.hd * es;
  g.ld = ld;
  g.k_cache = st.keys;
  g.v_cache = st.values;
  g.gate = gate;
  g.ld_gate = ld_gate;
  g.out = out.p;
  g.ldo = out.ld;
  g.out_mb = mb;
  g.fused = msa_grouped_fuses(&g, &b);
  if (!dry && !g.fused) HY(msa_grouped_rotate(&g, &b, stream));
  for (int s = 0; s < b.nseg;) {
    auto count = [&](int i) { return b.max_count == 1 ? 1 : b.host_start[i + 1] - b.host_start[i]; };
    const bool single = count(s) == 1;
    int e = b.max_count == 1 ? b.nseg : s + 1, longest = count(s);
    while (e < b.nseg && (count(e) == 1) == single) {
      longest = count(e) > longest ? count(e) : longest;
      ++e;
    }
    const int64_t save = off;
    g.splits = single ? msa_grouped_attention_splits(&g, e - s, b.key_bound) : 1;
    g.partial = g.splits > 1 ? (float*)alloc((int64_t)(e - s) * t.heads * g.splits * (t.vd + 4) * 4)
                             : nullptr;
    if (!dry) HY(msa_grouped_attention(&g, &b, s, e, longest, stream));
    off = save;
    s = e;
  }
  if (!dry && !g.fused) HY(msa_grouped_append(&g, &b, stream));
  return zero_tail(out, t.heads * t.vd);
}

int Run::parallel(int ri, const Act& h, Act& left, Act& right) {
  const msa_hybrid_layer& l = d->layers[d->runs[ri].layer];
  const msa_attention_layer& t = l.att;
  const int n_att = (t.heads + t.kv_heads) * t.hd + t.kv_heads * t.vd;
  const int C = 2 * l.kv_heads * l.dp + l.heads * l.vp, n2 = n_att + C, n32 = n2 + l.lr;
  const int n_gate = l.heads * l.vp, n_decay = l.heads * l.dp;
  char* in = (char*)alloc((int64_t)M * n2 * es);
  Act low = act(l.lr);
  float* z = (float*)alloc((int64_t)M * (l.n_in - n32) * 4);
  HY(linear_post(h, l.w_in, l.n_in, n32, l.in_bias, MSA_ACT_NONE, nullptr, in, false, &low, z));
  char* gate = (char*)alloc((int64_t)M * n_gate * es);
  float* decay = (float*)alloc((int64_t)M * n_decay * 4);
  HY(linear_post(low, l.w_lr, n_gate + n_decay, n_gate, l.lr_bias, MSA_ACT_NONE, l.lr_rate, gate, false,
                 nullptr, decay));
  const msa_hybrid_state st = dry ? msa_hybrid_state{} : a->state[ri];
  HY(grouped(l, st, in, n2, z, l.n_in - n32, left));
  msa_delta_args g{};
  g.ba = z + t.heads;
  g.ldba = l.n_in - n32;
  g.decay = decay;
  g.gate_act = MSA_GATE_SIGMOID;
  g.gate = gate;
  g.ld_gate = n_gate;
  return delta_core(l, st, in + (int64_t)n_att * es, n2, g, right);
}

// t arrives with everything that does not depend on the feed-forward
int Run::feed_forward(const msa_hybrid_layer& l, msa_tail_args& t) {
  const msa_hybrid_config& c = d->cfg;
  const Act h{t.h, c.Dp, c.Dp};
  int rc;
  if (l.ff_kind == MSA_FF_DENSE) {
    Act u = act(l.ff);
    HY(linear(h, l.w_ff_in, u.p, true, nullptr, l.n_ff_in, l.n_ff_in, MSA_GLU_GELU, 0.f));
    t.part = partial(u, l.w_ff_down, c.Dp, t.S, rc);
    HY(rc);
    return tail(t);
  }
  if (l.ff_kind == MSA_FF_RELU2) {
    Act u = act(l.ff);
    HY(linear_post(h, l.w_ff_in, l.n_ff_in, l.n_ff_in, l.ff_bias, MSA_ACT_RELU2, nullptr, u.p, true,
                   nullptr, nullptr));
    t.part = partial(u, l.w_ff_down, c.Dp, t.S, rc);
    HY(rc);
    t.bias = l.ff_down_bias;
    return tail(t);
  }
  const int n32 = 2 * l.ff_shared, ldz = l.n_ff_in - n32, E = l.experts, P = M * l.top;
  const bool shared = l.ff_shared > 0;
  Act u = shared ? act(l.ff_shared) : Act{};
  float* z = (float*)alloc((int64_t)M * ldz * 4);
  // the shared expert's hidden layer, the router logits and the shared gate's logit in one product
  HY(linear(h, l.w_ff_in, u.p, true, z, l.n_ff_in, n32, shared ? MSA_GLU_CLAMPED : MSA_GLU_NONE,
            l.limit_shared));
  const int avg = P / E, tile_rows = f32 ? 64 : avg <= 16 ? 16 : avg <= 32 ? 32
                                                 : avg <= 64 || mb > 0 ? 64 : 256;
  const int max_tiles = P / tile_rows + (E < P ? E : P);
  int32_t* ids = (int32_t*)alloc((int64_t)P * 4);
  float* w = (float*)alloc((int64_t)P * 4);
  float* sg = shared ? (float*)alloc((int64_t)M * 4) : nullptr;
  int32_t* perm = (int32_t*)alloc((int64_t)P * 4);
  int32_t* inverse = (int32_t*)alloc((int64_t)P * 4);
  int32_t* group_end = (int32_t*)alloc((int64_t)E * 4);
  int32_t* tile_group = (int32_t*)alloc((int64_t)max_tiles * 4);
  int32_t* tile_row = (int32_t*)alloc((int64_t)max_tiles * 4);
  int32_t* n_tiles = (int32_t*)alloc(4);
  void* eh = alloc((int64_t)P * l.ff_expert * es);
  void* ey = alloc((int64_t)P * c.Dp * es);
  if (!dry) {
    HY(msa_moe_route(z, ldz, M, E, l.n_groups, l.keep, l.top, l.router_scale, ids, w, sg, stream));
    HY(msa_moe_plan(ids, P, E, tile_rows, perm, inverse, group_end, tile_group, tile_row, n_tiles,
                    max_tiles, stream));
    msa_group_linear_args g{};
    g.dtype = c.dtype;
    g.groups = E;
    g.M = P;
    g.tile_group = tile_group;
    g.tile_row = tile_row;
    g.n_tiles = n_tiles;
    g.group_end = group_end;
    g.max_tiles = max_tiles;
    g.tile_rows = tile_rows;
    g.x = h.p;
    g.ldx = c.Dp;
    g.x_mb = mb;
    g.perm = perm;
    g.rows_per_x = l.top;
    g.W = l.w_e_in;
    g.y = eh;
    g.ldy = l.ff_expert;
    g.N = 2 * l.ff_expert;
    g.K = c.Dp;
    g.glu = MSA_GLU_CLAMPED;
    g.limit = l.limit_expert;
    HY(msa_group_linear(&g, stream));
    g.x = eh;
    g.ldx = l.ff_expert;
    g.x_mb = 0;
    g.perm = nullptr;
    g.W = l.w_e_down;
    g.y = ey;
    g.ldy = c.Dp;
    g.N = c.Dp;
    g.K = l.ff_expert;
    g.glu = MSA_GLU_NONE;
    HY(msa_group_linear(&g, stream));
  }
  if (shared) {
    t.part = partial(u, l.w_ff_down, c.Dp, t.S, rc);
    HY(rc);
    t.gate = sg;
  }
  t.top = l.top;
  t.pair_w = w;
  t.pair_y = ey;
  t.inverse = inverse;
  return tail(t);
}

int Run::go() {
  const msa_hybrid_config& c = d->cfg;
  const msa_batch& b = a->batch;
  float* x = (float*)alloc((int64_t)M * c.Dp * 4);
  float* e = d->adds_embedding ? (float*)alloc((int64_t)M * c.Dp * 4) : nullptr;
  Act h = act(c.Dp);
  auto step = [&](int pass) { return pass >= 0 ? c.loop_step + (int64_t)pass * c.Dp : nullptr; };
  if (!dry)
    HY(msa_embed_rmsnorm(c.dtype, a->tokens, b.tok_pos, M, c.embed, c.vocab, c.embed_scale, c.inv_freq,
                         c.D, c.Dp, c.eps, step(d->runs[0].pass), e, x,
                         d->layers[d->runs[0].layer].norm1, h.p, mb, stream));
  const int64_t layer_base = off;
  for (int i = 0; i < c.n_runs; ++i) {
    const msa_hybrid_layer& l = d->layers[d->runs[i].layer];
    const bool last = i + 1 == c.n_runs, ff = l.ff_kind != MSA_FF_NONE;
    // what ends the run: its output, what the loop adds, the next run's norm
    msa_tail_args end{};
    end.w_next = last ? c.final_norm : d->layers[d->runs[i + 1].layer].norm1;
    end.probe = a->probe ? a->probe + (int64_t)i * M * c.Dp : nullptr;
    const int pass = last ? -1 : d->runs[i + 1].pass;
    end.step = step(pass);
    end.add = pass > 0 ? e : nullptr;
    msa_tail_args t = ff ? msa_tail_args{} : end;
    if (ff) t.w_next = l.norm2;
    for (msa_tail_args* k : {&t, &end}) {
      k->dtype = c.dtype;
      k->M = M;
      k->D = c.D;
      k->Dp = c.Dp;
      k->eps = c.eps;
      k->x = x;
      k->h = h.p;
      k->h_mb = mb;
    }
    off = layer_base;
    const bool two = l.kind == MSA_MIX_PARALLEL, merged = two && !l.att.w_out;
    const Act both = act(merged ? 2 * l.ko : l.ko);
    Act o = merged ? columns(both, 0, l.ko) : both, o2{};
    t.w_post = l.norm1b;
    if (two) {
      o2 = merged ? columns(both, l.ko, l.ko) : act(l.att.ko);
      HY(parallel(i, h, o2, o));
      t.w_post = l.out_norm;
      t.w_post2 = l.att.out_norm;
    } else {
      HY(l.kind == MSA_MIX_LATENT ? latent(i, h, o) : l.kind == MSA_MIX_RGLRU ? rglru(i, h, o)
                                                                              : delta(i, h, o));
    }
    int rc;
    t.part = partial(both, l.w_out, c.Dp, t.S, rc, merged ? 2 : 1);
    HY(rc);
    if (merged) {
      t.S2 = t.S /= 2;
      t.part2 = t.part + (int64_t)t.S * M * c.Dp;
    } else if (two) {
      t.part2 = partial(o2, l.att.w_out, c.Dp, t.S2, rc);
      HY(rc);
    }
    HY(tail(t));
    off = layer_base;
    if (ff) {
      end.w_post = l.norm2b;
      HY(feed_forward(l, end));
    }
  }
  off = layer_base;
  if (!a->logits) return MSA_OK;
  Act f = h;
  int rows = M, fmb = mb;
  if (a->rows) {
    rows = a->n_rows;
    fmb = !f32 && rows <= MSA_PACKED_MAX_ROWS ? packed_row_blocks(rows) : 0;
    f = {alloc((int64_t)(fmb > 0 ? fmb * 16 : rows) * c.Dp * es), c.Dp, c.Dp};
    if (!dry) HY(msa_gather_rows(c.dtype, h.p, mb, a->rows, rows, c.Dp, f.p, fmb, stream));
  }
  if (dry || rows == 0) return MSA_OK;
  if (f32)
    return msa_linear_f32((const float*)f.p, (const float*)c.head, nullptr, a->logits, rows, c.Vp, c.Dp,
                          0, MSA_GLU_NONE, 0.f, stream);
  return msa_linear_partial_bf16(f.p, c.head, a->logits, rows, c.Vp, c.Dp, 1,
                                 fmb > 0 ? MSA_IN_PACKED : 0u, stream);
}

int start(Run& r, const msa_hybrid* d, const msa_hybrid_step_args* a, void* stream, bool dry) {
  const char* name = "msa_hybrid_step";
  MSA_REQUIRE(d && a, MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  const msa_batch& b = a->batch;
  MSA_REQUIRE(b.M > 0 && b.nseg > 0 && b.nseg <= b.M && b.max_count > 0 && b.key_bound > 0,
              MSA_ERR_INVALID_ARG, "%s: M=%d nseg=%d max_count=%d key_bound=%d", name, b.M, b.nseg,
              b.max_count, b.key_bound);
  MSA_REQUIRE(b.M <= 65535 && b.nseg <= 65535, MSA_ERR_CAPACITY, "%s: %d tokens in one call (65535)",
              name, b.M);
  MSA_REQUIRE(b.max_count == 1 ? b.nseg == b.M : (b.host_start && b.host_pos && b.host_slot),
              MSA_ERR_INVALID_ARG, "%s: segments of several tokens need host tables", name);
  if (b.host_start) {
    int longest = 0;
    for (int s = 0; s < b.nseg; ++s) {
      const int n = b.host_start[s + 1] - b.host_start[s];
      MSA_REQUIRE(n > 0 && n <= b.max_count, MSA_ERR_INVALID_ARG, "%s: segment %d holds %d tokens", name,
                  s, n);
      MSA_REQUIRE(b.host_pos[s] < 0 || (b.host_pos[s] + n <= a->capacity &&
                                        b.host_pos[s] + n <= b.key_bound),
                  MSA_ERR_CAPACITY, "%s: segment %d ends at position %d of %d", name, s,
                  b.host_pos[s] + n, a->capacity);
      if (n > longest) longest = n;
    }
    MSA_REQUIRE(b.host_start[0] == 0 && b.host_start[b.nseg] == b.M && longest == b.max_count,
                MSA_ERR_INVALID_ARG, "%s: the segments do not cover the batch", name);
  }
  r.d = d;
  r.a = a;
  r.stream = stream;
  r.dry = dry;
  r.f32 = d->cfg.dtype == MSA_F32;
  r.M = b.M;
  r.mb = !r.f32 && b.M <= MSA_PACKED_MAX_ROWS ? packed_row_blocks(b.M) : 0;
  r.es = r.f32 ? 4 : 2;
  r.base = dry ? nullptr : (char*)a->workspace;
  r.off = r.peak = 0;
  return MSA_OK;
}

}  // namespace

extern "C" int msa_hybrid_create(const msa_hybrid_config* cfg, const msa_hybrid_layer* layers,
                                 msa_hybrid** out) {
  const char* name = "msa_hybrid_create";
  MSA_REQUIRE(cfg && layers && out, MSA_ERR_INVALID_ARG, "%s: null pointer", name);
  MSA_REQUIRE((cfg->dtype == MSA_BF16 || cfg->dtype == MSA_F32) && cfg->layers > 0 && cfg->D > 0 &&
                  cfg->D <= cfg->Dp && cfg->Dp % 64 == 0 && cfg->Dp >= 128 && cfg->Dp <= 16384 &&
                  cfg->vocab > 0 && cfg->Vp % 16 == 0 && cfg->vocab <= cfg->Vp,
              MSA_ERR_INVALID_ARG, "%s: bad configuration", name);
  MSA_REQUIRE(cfg->embed && cfg->final_norm && cfg->head, MSA_ERR_INVALID_ARG,
              "%s: null pointer in the configuration", name);
  auto k_ok = [](int k) { return k >= 128 && k % 64 == 0; };
  for (int i = 0; i < cfg->layers; ++i) {
    const msa_hybrid_layer& l = layers[i];
    MSA_REQUIRE(l.w_in && l.w_out && l.norm1 && k_ok(l.ko) && l.n_in % 16 == 0,
                MSA_ERR_INVALID_ARG, "%s: layer %d: mixer projections", name, i);
    if (l.kind == MSA_MIX_LATENT) {
      MSA_REQUIRE(k_ok(l.qp) && k_ok(l.rp) && l.rp <= 2048 && l.hd % 32 == 0 && l.heads > 0 &&
                      l.ko >= l.heads * l.hd && l.w_q && l.w_absorb && l.w_v && l.wq_norm &&
                      (cfg->dtype == MSA_F32 || l.w_kv) && l.scale > 0.f &&
                      l.n_in >= l.qp + (l.kv_from < 0 ? l.rp : 0),
                  MSA_ERR_INVALID_ARG, "%s: layer %d: latent attention", name, i);
      MSA_REQUIRE(l.kv_from < i && (l.kv_from >= 0 ? layers[l.kv_from].kind == MSA_MIX_LATENT &&
                                                         layers[l.kv_from].kv_from < 0 &&
                                                         layers[l.kv_from].rp == l.rp
                                                   : l.wkv_norm != nullptr),
                  MSA_ERR_INVALID_ARG, "%s: layer %d: no latent at layer %d", name, i, l.kv_from);
    } else if (l.kind == MSA_MIX_RGLRU) {
      MSA_REQUIRE(l.channels > 0 && l.blocks > 0 && l.channels % (32 * l.blocks) == 0 &&
                      l.n_in == 2 * l.channels && l.ko >= l.channels && l.w_gates && l.conv_w &&
                      l.gate_bias && l.lam && l.y_bias,
                  MSA_ERR_INVALID_ARG, "%s: layer %d: gated linear recurrent unit", name, i);
    } else if (l.kind == MSA_MIX_PARALLEL) {
      const msa_attention_layer& t = l.att;
      MSA_REQUIRE(t.heads > 0 && t.kv_heads > 0 && t.heads % t.kv_heads == 0 && t.hd > 0 &&
                      t.hd % 16 == 0 && t.vd > 0 && t.vd % 16 == 0 && t.chunk >= 0 && t.scale > 0.f &&
                      (t.rot_dims == 0 || t.inv_freq) && t.out_norm && k_ok(t.ko) &&
                      (t.w_out || (t.ko == l.ko && cfg->dtype == MSA_BF16)) &&
                      t.ko >= t.heads * t.vd,
                  MSA_ERR_INVALID_ARG, "%s: layer %d: grouped attention", name, i);
      MSA_REQUIRE(l.heads > 0 && l.kv_heads > 0 && l.heads % l.kv_heads == 0 && l.conv_w && l.o_norm &&
                      l.ko >= l.heads * l.vp && l.vp <= 512 && k_ok(l.lr) && l.w_lr && l.lr_bias &&
                      l.lr_rate && l.out_norm && l.in_bias &&
                      l.n_in >= (t.heads + t.kv_heads) * t.hd + t.kv_heads * t.vd +
                                    2 * l.kv_heads * l.dp + l.heads * l.vp + l.lr + t.heads + l.heads,
                  MSA_ERR_INVALID_ARG, "%s: layer %d: delta rule beside attention", name, i);
    } else {
      MSA_REQUIRE(l.kind == MSA_MIX_DELTA && l.heads > 0 && l.kv_heads > 0 &&
                      l.heads % l.kv_heads == 0 && l.conv_w && l.decay_rate && l.dt_bias && l.o_norm &&
                      l.ko >= l.heads * l.vp && l.vp <= 512 &&
                      l.n_in >= 2 * l.kv_heads * l.dp + 2 * l.heads * l.vp + 2 * l.heads,
                  MSA_ERR_INVALID_ARG, "%s: layer %d: gated delta rule", name, i);
    }
    if (l.ff_kind == MSA_FF_DENSE)
      MSA_REQUIRE(k_ok(l.ff) && l.n_ff_in == 2 * l.ff && l.w_ff_in && l.w_ff_down && l.norm2,
                  MSA_ERR_INVALID_ARG, "%s: layer %d: feed-forward", name, i);
    else if (l.ff_kind == MSA_FF_RELU2)
      MSA_REQUIRE(k_ok(l.ff) && l.n_ff_in == l.ff && l.w_ff_in && l.w_ff_down && l.norm2,
                  MSA_ERR_INVALID_ARG, "%s: layer %d: feed-forward", name, i);
    else if (l.ff_kind == MSA_FF_MOE)
      MSA_REQUIRE(l.experts > 0 && l.top > 0 && k_ok(l.ff_expert) && l.w_ff_in &&
                      l.w_e_in && l.w_e_down && l.norm2 && l.n_groups > 0 &&
                      (l.ff_shared == 0 || (k_ok(l.ff_shared) && l.w_ff_down)) &&
                      l.n_ff_in >= 2 * l.ff_shared + l.experts + (l.ff_shared > 0 ? 1 : 0),
                  MSA_ERR_INVALID_ARG, "%s: layer %d: routed feed-forward", name, i);
  }
  const int n_runs = cfg->n_runs > 0 ? cfg->n_runs : cfg->layers;
  MSA_REQUIRE(cfg->n_runs <= 0 || (cfg->run_layer && cfg->run_pass), MSA_ERR_INVALID_ARG,
              "%s: runs without tables", name);
  msa_hybrid* d = new (std::nothrow) msa_hybrid();
  msa_hybrid_layer* lw = (msa_hybrid_layer*)malloc(sizeof(msa_hybrid_layer) * (size_t)cfg->layers);
  LayerRun* runs = (LayerRun*)malloc(sizeof(LayerRun) * (size_t)n_runs);
  auto drop = [&] {
    delete d;
    free(lw);
    free(runs);
  };
  if (!d || !lw || !runs) {
    drop();
    msa_set_error("%s: out of host memory", name);
    return MSA_ERR_INVALID_ARG;
  }
  for (int i = 0; i < n_runs; ++i) {
    LayerRun& r = runs[i];
    r.layer = cfg->n_runs > 0 ? cfg->run_layer[i] : i;
    r.pass = cfg->n_runs > 0 ? cfg->run_pass[i] : -1;
    r.owner = i;
    bool ok = r.layer >= 0 && r.layer < cfg->layers && (r.pass < 0 || cfg->loop_step);
    if (ok && layers[r.layer].kind == MSA_MIX_LATENT && layers[r.layer].kv_from >= 0) {
      // the latest run of the layer that owns the latent
      for (r.owner = i - 1; r.owner >= 0 && runs[r.owner].layer != layers[r.layer].kv_from;) --r.owner;
      ok = r.owner >= 0;
    }
    if (!ok) {
      drop();
      msa_set_error("%s: run %d", name, i);
      return MSA_ERR_INVALID_ARG;
    }
    if (r.pass > 0) d->adds_embedding = true;
  }
  memcpy(lw, layers, sizeof(msa_hybrid_layer) * (size_t)cfg->layers);
  d->cfg = *cfg;
  d->layers = lw;
  d->runs = runs;
  d->cfg.n_runs = n_runs;
  d->cfg.run_layer = d->cfg.run_pass = nullptr;
  *out = d;
  return MSA_OK;
}

extern "C" void msa_hybrid_destroy(msa_hybrid* d) {
  if (!d) return;
  free(d->layers);
  free(d->runs);
  delete d;
}

extern "C" int64_t msa_hybrid_workspace_bytes(const msa_hybrid* d, const msa_hybrid_step_args* a) {
  Run r{};
  if (start(r, d, a, nullptr, true) || r.go()) return 0;
  return r.peak;
}

extern "C" int msa_hybrid_step(const msa_hybrid* d, const msa_hybrid_step_args* a, void* stream) {
  const char* name = "msa_hybrid_step";
  Run r{};
  HY(start(r, d, a, stream, true));
  HY(r.go());
  const int64_t need = r.peak;
  const msa_batch& b = a->batch;
  MSA_REQUIRE(a->tokens && a->state && a->workspace && b.tok_slot && b.tok_pos && b.tok_off &&
                  b.seg_start && b.seg_slot && b.seg_pos && a->capacity > 0,
              MSA_ERR_INVALID_ARG, "%s: null pointer in the step's arguments", name);
  MSA_REQUIRE(a->workspace_bytes >= need, MSA_ERR_CAPACITY, "%s: workspace of %lld bytes, %lld needed",
              name, (long long)a->workspace_bytes, (long long)need);
  for (int i = 0; i < d->cfg.n_runs; ++i) {
    const msa_hybrid_layer& l = d->layers[d->runs[i].layer];
    const msa_hybrid_state& st = a->state[i];
    MSA_REQUIRE(l.kind == MSA_MIX_LATENT ? (l.kv_from >= 0 || st.latent)
                                         : (st.rec && (st.conv || l.taps == 1)),
                MSA_ERR_INVALID_ARG, "%s: run %d has no cache or state", name, i);
    const int rows = l.att.chunk > 0 && l.att.chunk < a->capacity ? l.att.chunk : a->capacity;
    MSA_REQUIRE(l.kind != MSA_MIX_PARALLEL || (st.keys && st.values && st.kv_rows >= rows),
                MSA_ERR_INVALID_ARG, "%s: run %d keeps %d positions of %d", name, i, st.kv_rows, rows);
  }
  HY(start(r, d, a, stream, false));
  return r.go();
}
