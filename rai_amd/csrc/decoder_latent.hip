// Driver of the latent-attention decoders (RAI_ARCH_LELITAR): a parallel block over an f32 residual stream,
//   x <- x + m * (attention(n1(x)) + mlp(n2(x))),
// every layer with sizes of its own, the MLP dense, a mixture of experts or absent.
//
// Per layer, in a prefill:
//   stream norm (adds the previous mixture's outputs, writes both norms' rows)
//   Wd . h1 -> [query latent | latent | gate], norms of the latents, cache append
//   Wuq . cq -> q;  Wkv . c -> k | v of the visible context;  flash attention with window and output gate
//   dense:   gate|up . h2 with the gated epilogue, then [o | down] as one contraction with the f32 residual epilogue
//   mixture: o with the residual epilogue, router logits, plan, scaled gather, two grouped products; the sum over a
//            token's experts waits for the next stream norm
// Fewer than kAbsorbRows new tokens per sequence take the absorbed attention over the cached latents instead of the
// expansion.  Only the normalised latents are cached.
#include <cmath>

#include "decoder.h"

namespace rai {

constexpr int kAbsorbRows = 16;   // the flash kernel serves 16 query rows and more

// Device memory that starts as zeros: padding rows and columns are never written by a loader.
int zalloc(rai_hip_decoder *d, size_t bytes, char **out) {
  RAI_TRY(dalloc(d, bytes, out));
  RAI_HIP_TRY(hipMemset(*out, 0, bytes ? bytes : 16));
  return RAI_OK;
}

// Rows (columns) in groups of `group`, each padded to `stride` elements.
void add_grouped_slot(rai_hip_decoder *d, const std::string &name, int64_t rows, int64_t cols, char *dst, int64_t pitch,
                      int64_t row_group, int64_t row_stride, int64_t col_group, int64_t col_stride) {
  add_slot(d, name, rows, cols, dst, pitch);
  ParamSlot &s = d->slots.back();
  s.row_group = row_group; s.row_stride = row_stride;
  s.col_group = col_group; s.col_stride = col_stride;
}

static int create_layer(rai_hip_decoder *d, int l, const rai_hip_latent_layer &c) {
  LatentModel &lm = *d->latent;
  LatentLayer y;
  memset(&y, 0, sizeof(y));
  y.c = c;
  const size_t es = d->es;
  const int H = d->H, Hp = lm.Hp;
  y.Qp = pad64(c.q_rank);
  y.Rp = pad64(c.kv_rank);
  y.Dp = pad_head(c.qk_dim > c.v_dim ? c.qk_dim : c.v_dim);
  y.QD = c.heads * y.Dp;
  y.ldn = y.Qp + y.Rp + y.QD;
  const bool dense = c.mlp_kind == RAI_MLP_DENSE, moe = c.mlp_kind == RAI_MLP_MIXTURE;
  y.Fp = dense ? pad64(c.intermediate) : 0;
  y.EFp = moe ? pad64(c.intermediate) : 0;
  const int KB = y.QD + y.Fp;
  RAI_TRY(zalloc(d, (size_t)H * es, &y.n1_w));
  RAI_TRY(zalloc(d, (size_t)c.q_rank * es, &y.q_w));
  RAI_TRY(zalloc(d, (size_t)c.kv_rank * es, &y.c_w));
  RAI_TRY(zalloc(d, (size_t)y.ldn * Hp * es, &y.Wd));
  RAI_TRY(zalloc(d, (size_t)y.QD * y.Qp * es, &y.Wuq));
  RAI_TRY(zalloc(d, (size_t)2 * y.QD * y.Rp * es, &y.Wkv));
  RAI_TRY(zalloc(d, (size_t)y.QD * y.Rp * es, &y.WukT));
  RAI_TRY(zalloc(d, (size_t)Hp * KB * es, &y.Wb));
  RAI_TRY(zalloc(d, (size_t)d->cfg.max_batch * d->cfg.max_context * y.Rp * es, &y.cache));
  const std::string p = "l" + std::to_string(l) + ".", mix = p + "mix.", mlp = p + "mlp.";
  add_slot(d, p + "norm1", 1, H, y.n1_w, H);
  add_slot(d, mix + "dq", c.q_rank, H, y.Wd, Hp);
  add_slot(d, mix + "dq.norm", 1, c.q_rank, y.q_w, c.q_rank);
  add_grouped_slot(d, mix + "uq", (int64_t)c.heads * c.qk_dim, c.q_rank, y.Wuq, y.Qp, c.qk_dim, (int64_t)y.Dp * y.Qp, 0, 0);
  add_slot(d, mix + "dkv", c.kv_rank, H, y.Wd + (size_t)y.Qp * Hp * es, Hp);
  add_slot(d, mix + "dkv.norm", 1, c.kv_rank, y.c_w, c.kv_rank);
  add_grouped_slot(d, mix + "uk", (int64_t)c.heads * c.qk_dim, c.kv_rank, y.Wkv, y.Rp, c.qk_dim, (int64_t)y.Dp * y.Rp, 0, 0);
  add_grouped_slot(d, mix + "uv", (int64_t)c.heads * c.v_dim, c.kv_rank, y.Wkv + (size_t)y.QD * y.Rp * es, y.Rp, c.v_dim,
                   (int64_t)y.Dp * y.Rp, 0, 0);
  add_grouped_slot(d, mix + "g", (int64_t)c.heads * c.v_dim, H, y.Wd + (size_t)(y.Qp + y.Rp) * Hp * es, Hp, c.v_dim,
                   (int64_t)y.Dp * Hp, 0, 0);
  add_grouped_slot(d, mix + "o", H, (int64_t)c.heads * c.v_dim, y.Wb, KB, 0, 0, c.v_dim, y.Dp);
  if (dense || moe) {
    RAI_TRY(zalloc(d, (size_t)H * es, &y.n2_w));
    add_slot(d, p + "norm2", 1, H, y.n2_w, H);
  }
  if (dense) {
    RAI_TRY(zalloc(d, (size_t)2 * y.Fp * Hp * es, &y.Wgu));
    add_slot(d, mlp + "gate", c.intermediate, H, y.Wgu, 2 * (int64_t)Hp);
    add_slot(d, mlp + "up", c.intermediate, H, y.Wgu + (size_t)Hp * es, 2 * (int64_t)Hp);
    add_slot(d, mlp + "down", H, c.intermediate, y.Wb + (size_t)y.QD * es, KB);
  }
  if (moe) {
    const size_t gu = (size_t)2 * y.EFp * Hp, dn = (size_t)Hp * y.EFp;
    RAI_TRY(zalloc(d, (size_t)c.experts * Hp * es, &y.Wr));
    RAI_TRY(zalloc(d, c.experts * gu * es, &y.We_gu));
    RAI_TRY(zalloc(d, c.experts * dn * es, &y.We_dn));
    add_slot(d, mlp + "router", c.experts, H, y.Wr, Hp);
    for (int e = 0; e < c.experts; ++e) {
      const std::string q = mlp + "e" + std::to_string(e) + ".";
      add_slot(d, q + "gate", c.intermediate, H, y.We_gu + e * gu * es, 2 * (int64_t)Hp);
      add_slot(d, q + "up", c.intermediate, H, y.We_gu + (e * gu + Hp) * es, 2 * (int64_t)Hp);
      add_slot(d, q + "down", H, c.intermediate, y.We_dn + e * dn * es, y.EFp);
    }
  }
  lm.layers.push_back(y);
  return RAI_OK;
}

static int create_latent(rai_hip_decoder *d, const rai_hip_latent_config &cfg, const rai_hip_latent_layer *layers) {
  LatentModel &lm = *d->latent;
  const size_t es = d->es;
  const int H = d->H, Hp = lm.Hp = pad64(H), V = d->V;
  RAI_TRY(decoder_alloc_common(d));
  RAI_TRY(zalloc(d, (size_t)V * H * es, &d->embed));
  add_slot(d, "embed", V, H, d->embed, H);
  for (int l = 0; l < cfg.num_layers; ++l) RAI_TRY(create_layer(d, l, layers[l]));
  RAI_TRY(zalloc(d, (size_t)H * es, &d->lnf_w));
  add_slot(d, "final.norm", 1, H, d->lnf_w, H);
  RAI_TRY(zalloc(d, (size_t)V * Hp * es, &d->head_w));
  add_slot(d, "head", V, H, d->head_w, Hp);
  d->head_b = nullptr;

  // activations, sized for the widest layer
  int Qp = 0, Rp = 0, QD = 0, ldn = 0, KB = 0, EFp = 0, experts = 0;
  size_t ws = 0;
  int64_t top = 0, tiles = 0, counts = 0;
  const int64_t rows = d->max_rows;
  const int64_t absorb_rows = std::min<int64_t>(rows, (int64_t)cfg.max_batch * (kAbsorbRows - 1));
  size_t qa = 0;
  const int bm = cfg.dtype == RAI_BF16 ? kGroupedRowsBf16 : kGroupedRowsF32;
  for (const LatentLayer &y : lm.layers) {
    Qp = std::max(Qp, y.Qp); Rp = std::max(Rp, y.Rp); QD = std::max(QD, y.QD);
    ldn = std::max(ldn, y.ldn); KB = std::max(KB, y.QD + y.Fp); EFp = std::max(EFp, y.EFp);
    ws = std::max(ws, latent_attn_ws_floats((int)absorb_rows, y.c.heads, y.Rp));
    qa = std::max(qa, (size_t)absorb_rows * y.c.heads * y.Rp);
    if (y.c.mlp_kind == RAI_MLP_MIXTURE) {
      experts = std::max(experts, y.c.experts);
      top = std::max<int64_t>(top, y.c.top);
      tiles = std::max<int64_t>(tiles, moe_max_tiles(rows * y.c.top, y.c.experts, bm));
      counts = std::max(counts, moe_plan_counts(rows * y.c.top, y.c.experts));
    }
  }
  char *tmp = nullptr;
  RAI_TRY(zalloc(d, rows * H * es, &d->x));
  RAI_TRY(zalloc(d, rows * Hp * sizeof(float), &tmp));
  lm.xs = (float *)tmp;
  RAI_TRY(zalloc(d, rows * Hp * es, &lm.h1));
  RAI_TRY(zalloc(d, rows * Hp * es, &lm.h2));
  RAI_TRY(zalloc(d, rows * ldn * es, &lm.dn));
  RAI_TRY(zalloc(d, rows * Qp * es, &lm.cq));
  RAI_TRY(zalloc(d, rows * Rp * es, &lm.cn));
  RAI_TRY(zalloc(d, rows * QD * es, &lm.q));
  // the expanded keys and values of a prefill; the absorbed form keeps its latent-space queries there
  RAI_TRY(zalloc(d, std::max((size_t)rows * 2 * QD, qa) * es, &lm.kv));
  RAI_TRY(zalloc(d, rows * KB * es, &lm.cat));
  RAI_TRY(zalloc(d, (size_t)cfg.max_batch * Hp * es, &d->last));
  RAI_TRY(zalloc(d, ws * sizeof(float), &tmp));
  lm.ws = (float *)tmp;
  if (experts) {
    const int64_t slots = rows * top;
    RAI_TRY(zalloc(d, slots * Hp * es, &lm.gathered));
    RAI_TRY(zalloc(d, slots * EFp * es, &lm.eact));
    RAI_TRY(zalloc(d, slots * Hp * es, &lm.eout));
    RAI_TRY(zalloc(d, rows * experts * sizeof(float), &tmp));
    lm.rlogits = (float *)tmp;
    RAI_TRY(zalloc(d, slots * sizeof(float), &tmp));
    lm.rweight = (float *)tmp;
    RAI_TRY(zalloc(d, slots * sizeof(int), &tmp));
    lm.rchoice = (int *)tmp;
    RAI_TRY(zalloc(d, slots * sizeof(int), &tmp));
    lm.rpos = (int *)tmp;
    RAI_TRY(zalloc(d, slots * sizeof(int), &tmp));
    lm.plan.slot_of = (int *)tmp;
    RAI_TRY(zalloc(d, counts * sizeof(int), &tmp));
    lm.plan.counts = (int *)tmp;
    RAI_TRY(zalloc(d, tiles * sizeof(int4), &tmp));
    lm.plan.tiles = (int4 *)tmp;
    RAI_TRY(zalloc(d, sizeof(int), &tmp));
    lm.plan.n_tiles = (int *)tmp;
    lm.plan.cap_tiles = (int)tiles;
  }
  return RAI_OK;
}

// ------------------------------------------------------------------ forward
static int ensure_derived(rai_hip_decoder *d, hipStream_t st) {
  LatentModel &lm = *d->latent;
  if (lm.derived_ready) return RAI_OK;
  for (LatentLayer &y : lm.layers)
    RAI_TRY(launch_latent_transpose_uk(st, d->cfg.dtype, y.Wkv, y.WukT, y.c.heads, y.Dp, y.Rp));
  lm.derived_ready = true;
  return RAI_OK;
}

static int ensure_latent_fragments(rai_hip_decoder *d, hipStream_t st) {
  LatentModel &lm = *d->latent;
  if (d->frag_ready) return RAI_OK;
  for (LatentLayer &y : lm.layers) {
    const int KB = y.QD + y.Fp;
    RAI_TRY(decoder_fragments(d, st, y.Wd, lm.Hp, y.ldn, lm.Hp, &y.Wd_f));
    RAI_TRY(decoder_fragments(d, st, y.Wuq, y.Qp, y.QD, y.Qp, &y.Wuq_f));
    RAI_TRY(decoder_fragments(d, st, y.Wgu, lm.Hp, 2 * y.Fp, lm.Hp, &y.Wgu_f));
    RAI_TRY(decoder_fragments(d, st, y.Wb, KB, lm.Hp, KB, &y.Wb_f));
    RAI_TRY(decoder_fragments(d, st, y.Wr, lm.Hp, y.c.experts, lm.Hp, &y.Wr_f));
  }
  RAI_TRY(decoder_fragments(d, st, d->head_w, lm.Hp, d->V, lm.Hp, &d->head_f));
  d->frag_ready = true;
  return RAI_OK;
}

static LinearArgs latent_linear_args(rai_hip_decoder *d, const void *A, int64_t lda, int64_t M, const char *W, int N, int K) {
  LinearArgs a = linear_args_default();
  a.A = A; a.lda = lda;
  a.W = W; a.ldw = K;
  a.M = (int)M; a.N = N; a.K = K; a.n_split = N;
  a.splitk_ws = d->splitk_ws; a.splitk_ws_bytes = d->splitk_ws_bytes;
  return a;
}

// out = mult * A W^T + out, out the f32 stream
static int residual_linear(rai_hip_decoder *d, hipStream_t st, const void *A, int64_t lda, int64_t M, const char *W, int K, const char *Wfrag) {
  LatentModel &lm = *d->latent;
  LinearArgs a = latent_linear_args(d, A, lda, M, W, lm.Hp, K);
  a.ldw = lda;   // the activation buffer and the packed matrix have the same columns
  a.Wfrag = Wfrag;
  a.out1 = lm.xs; a.ld1 = lm.Hp;
  a.residual = lm.xs; a.ldr = lm.Hp;
  a.f32_out = 1; a.out_scale = (float)lm.c.residual_mult;
  return decoder_linear(d, st, a);
}

static int expanded_attention(rai_hip_decoder *d, hipStream_t st, const LatentLayer &y, int B, int S) {
  LatentModel &lm = *d->latent;
  const int dt = d->cfg.dtype, QD = y.QD, KB = QD + y.Fp;
  const size_t es = d->es;
  const int seen = y.c.window > 0 && y.c.window - 1 < d->ctx_len ? y.c.window - 1 : d->ctx_len;   // cached tokens in reach
  const int T = seen + S;
  auto expand = [&](const char *c, int64_t n, char *kv) -> int {
    LinearArgs a = latent_linear_args(d, c, y.Rp, n, y.Wkv, 2 * QD, y.Rp);
    a.out1 = kv; a.ld1 = 2 * QD;
    return decoder_linear(d, st, a);
  };
  if (seen == 0) {
    RAI_TRY(expand(lm.cn, (int64_t)B * S, lm.kv));
  } else {
    for (int b = 0; b < B; ++b)
      RAI_TRY(expand(y.cache + ((size_t)b * d->cfg.max_context + (d->ctx_len - seen)) * y.Rp * es, T, lm.kv + (size_t)b * T * 2 * QD * es));
  }
  AttnArgs t;
  memset(&t, 0, sizeof(t));
  t.q = lm.q; t.k = lm.kv; t.v = lm.kv + (size_t)QD * es;
  t.out = lm.cat; t.out_row_stride = KB;
  t.qs[0] = (int64_t)S * QD; t.qs[1] = y.Dp; t.qs[2] = QD;
  t.ks[0] = t.vs[0] = (int64_t)T * 2 * QD; t.ks[1] = t.vs[1] = y.Dp; t.ks[2] = t.vs[2] = 2 * QD;
  t.B = B; t.Hq = t.Hkv = y.c.heads; t.S = S; t.T = T; t.D = y.Dp;
  t.scale = (float)y.c.attn_scale;
  t.causal = 1; t.f32_scores = 1; t.dtype = dt;
  t.window = y.c.window;
  t.gate = lm.dn + (size_t)(y.Qp + y.Rp) * es; t.gate_row_stride = y.ldn;
  return launch_attention(st, t);
}

static int absorbed_attention(rai_hip_decoder *d, hipStream_t st, const LatentLayer &y, int B, int S) {
  LatentModel &lm = *d->latent;
  LatentAttnArgs t;
  memset(&t, 0, sizeof(t));
  t.q = lm.q; t.WukT = y.WukT; t.Wuv = y.Wkv + (size_t)y.QD * y.Rp * d->es;
  t.cache = y.cache;
  t.gate = lm.dn + (size_t)(y.Qp + y.Rp) * d->es; t.ldg = y.ldn;
  t.out = lm.cat; t.ldo = y.QD + y.Fp;
  t.qa = lm.kv; t.ws = lm.ws;
  t.state = d->state;
  t.B = B; t.S = S; t.heads = y.c.heads; t.Dp = y.Dp; t.Rp = y.Rp; t.Tmax = d->cfg.max_context; t.window = y.c.window;
  t.scale = (float)y.c.attn_scale;
  return launch_latent_attention(st, d->cfg.dtype, t);
}

// Adds the mixture to the stream when *pending comes back null; otherwise leaves the experts' outputs in lm.eout, row
// lm.rpos[token * top + j], for the next stream norm to add.
static int mixture(rai_hip_decoder *d, hipStream_t st, const LatentLayer &y, int64_t M, const LatentLayer **pending) {
  LatentModel &lm = *d->latent;
  const int dt = d->cfg.dtype, Hp = lm.Hp, top = y.c.top;
  LinearArgs r = latent_linear_args(d, lm.h2, Hp, M, y.Wr, y.c.experts, Hp);
  r.out1 = lm.rlogits; r.ld1 = y.c.experts;
  r.f32_out = 1; r.out_scale = 1.f;
  r.Wfrag = wants_fragments(d, M) ? y.Wr_f : nullptr;
  RAI_TRY(decoder_linear(d, st, r));
  RAI_TRY(launch_moe_route(st, lm.rlogits, M, y.c.experts, top, lm.rchoice, lm.rweight));
  const int64_t slots = M * top;
  const int64_t gs = (int64_t)2 * y.EFp * Hp, os = (int64_t)Hp * y.EFp;
  if (dt == RAI_BF16 && moe_slots_serves(slots, y.c.experts, Hp, top, y.EFp)) {
    MoeSlotsArgs m;
    memset(&m, 0, sizeof(m));
    m.h = lm.h2; m.ld = Hp; m.slots = (int)slots; m.top = top; m.choice = lm.rchoice; m.weight = lm.rweight;
    m.We_gu = y.We_gu; m.Hp = Hp; m.EFp = y.EFp; m.act = y.c.mlp_act; m.gu_stride = gs; m.eact = lm.eact;
    RAI_TRY(launch_moe_slots(st, m));
    LatentDownArgs dn;
    memset(&dn, 0, sizeof(dn));
    dn.x1 = lm.eact; dn.W1 = y.We_dn; dn.K1 = y.EFp; dn.top = top; dn.stride1 = os; dn.choice = lm.rchoice;
    dn.res = lm.xs; dn.res_f32 = 1; dn.H = d->H; dn.N = Hp; dn.rows = (int)M;
    dn.mult = (float)lm.c.residual_mult;
    dn.out = lm.xs;
    *pending = nullptr;
    return launch_latent_down(st, dn);
  }
  *pending = &y;
  const int bm = linear_grouped_rows(dt, slots, y.c.experts);
  MoePlan plan = lm.plan;
  plan.cap_tiles = moe_max_tiles(slots, y.c.experts, bm);
  RAI_TRY(launch_moe_plan(st, lm.rchoice, slots, y.c.experts, bm, plan, lm.rpos));
  RAI_TRY(launch_moe_gather(st, dt, lm.h2, Hp, Hp, plan, lm.rweight, top, slots, lm.gathered));
  LinearArgs g = latent_linear_args(d, lm.gathered, Hp, slots, y.We_gu, 2 * y.EFp, Hp);
  g.out1 = lm.eact; g.ld1 = y.EFp;
  g.act = y.c.mlp_act; g.act_from = 0; g.glu = 1;
  LinearArgs o = latent_linear_args(d, lm.eact, y.EFp, slots, y.We_dn, Hp, y.EFp);
  o.out1 = lm.eout; o.ld1 = Hp;
  if (dt == RAI_BF16) {
    RAI_TRY(launch_linear_bf16_grouped(st, g, gs, plan, bm));
    return launch_linear_bf16_grouped(st, o, os, plan, bm);
  }
  RAI_TRY(launch_linear_f32_grouped(st, g, gs, plan));
  return launch_linear_f32_grouped(st, o, os, plan);
}

static StreamNormArgs stream_norm_args(rai_hip_decoder *d, int64_t rows) {
  LatentModel &lm = *d->latent;
  StreamNormArgs n;
  memset(&n, 0, sizeof(n));
  n.src = lm.xs; n.src_f32 = 1; n.src_ld = lm.Hp;
  n.x_ld = lm.Hp; n.h_ld = lm.Hp;
  n.width = d->H; n.groups = lm.c.norm_groups; n.eps = (float)lm.c.norm_eps;
  n.rows = rows; n.first = 0; n.step = 1;
  return n;
}

// Adds the outputs a mixture left pending to the stream rows a norm is about to read (and writes the stream back).
static void add_pending(rai_hip_decoder *d, const LatentLayer *y, StreamNormArgs *n) {
  LatentModel &lm = *d->latent;
  if (!y) return;
  n->add = lm.eout; n->add_ld = lm.Hp; n->add_rows = lm.rpos; n->top = y->c.top;
  n->add_scale = (float)lm.c.residual_mult;
  n->x = lm.xs;
}

// One bf16 row: six launches a layer, nothing materialised between a norm and the product it feeds.
static bool single_row_ok(const rai_hip_decoder *d) {
  const LatentModel &lm = *d->latent;
  int rank = 0, experts = 0;
  int64_t cols = 0;
  for (const LatentLayer &y : lm.layers) {
    rank = std::max(rank, std::max(y.Qp, y.Rp));
    if (y.c.mlp_kind == RAI_MLP_MIXTURE) experts = std::max(experts, y.c.experts);
    cols = std::max<int64_t>(cols, y.QD + y.Fp + (int64_t)y.c.top * y.EFp);
  }
  return d->cfg.dtype == RAI_BF16 && latent_single_row_serves(d->H, lm.c.norm_groups, rank, experts, cols);
}

static int single_row_layers(rai_hip_decoder *d, hipStream_t st) {
  LatentModel &lm = *d->latent;
  const size_t es = d->es;
  for (int l = 0; l < d->L; ++l) {
    const LatentLayer &y = lm.layers[l];
    const bool dense = y.c.mlp_kind == RAI_MLP_DENSE, moe = y.c.mlp_kind == RAI_MLP_MIXTURE;
    const void *src = l == 0 ? (const void *)d->x : (const void *)lm.xs;
    LatentInArgs in;
    memset(&in, 0, sizeof(in));
    in.src = src; in.src_f32 = l > 0;
    in.H = d->H; in.groups = lm.c.norm_groups; in.K = lm.Hp; in.eps = (float)lm.c.norm_eps; in.ldw = lm.Hp;
    in.W1 = y.Wd; in.n1 = y.n1_w; in.N1 = y.ldn; in.out1 = lm.dn;
    in.n2 = y.n2_w; in.act = y.c.mlp_act;
    if (dense) { in.W2 = y.Wgu; in.N2 = 2 * y.Fp; in.gated2 = 1; in.out2 = lm.cat + (size_t)y.QD * es; }
    if (moe) { in.W2 = y.Wr; in.N2 = y.c.experts; in.out2 = lm.rlogits; in.h2 = lm.h2; }
    RAI_TRY(launch_latent_in(st, in));
    LatentMidArgs m;
    memset(&m, 0, sizeof(m));
    m.dn = lm.dn;
    m.q_rank = y.c.q_rank; m.Qp = y.Qp; m.kv_rank = y.c.kv_rank; m.Rp = y.Rp;
    m.q_w = y.q_w; m.c_w = y.c_w; m.eps = (float)lm.c.norm_eps;
    m.Wuq = y.Wuq; m.Nq = y.QD; m.q = lm.q;
    m.cache = y.cache; m.state = d->state;
    if (moe) {
      m.rlogits = lm.rlogits; m.experts = y.c.experts; m.top = y.c.top;
      m.h2 = lm.h2; m.We_gu = y.We_gu; m.Hp = lm.Hp; m.EFp = y.EFp; m.act = y.c.mlp_act;
      m.gu_stride = (int64_t)2 * y.EFp * lm.Hp;
      m.eact = lm.eact; m.choice = lm.rchoice;
    }
    RAI_TRY(launch_latent_mid(st, m));
    RAI_TRY(absorbed_attention(d, st, y, 1, 1));
    LatentDownArgs dn;
    memset(&dn, 0, sizeof(dn));
    dn.x0 = lm.cat; dn.W0 = y.Wb; dn.K0 = y.QD + y.Fp;
    if (moe) { dn.x1 = lm.eact; dn.W1 = y.We_dn; dn.K1 = y.EFp; dn.top = y.c.top; dn.stride1 = (int64_t)lm.Hp * y.EFp; dn.choice = lm.rchoice; }
    dn.res = src; dn.res_f32 = l > 0; dn.H = d->H; dn.N = lm.Hp; dn.rows = 1;
    dn.mult = (float)lm.c.residual_mult;
    dn.out = lm.xs;
    RAI_TRY(launch_latent_down(st, dn));
  }
  // final norm and head
  LatentInArgs h;
  memset(&h, 0, sizeof(h));
  h.src = lm.xs; h.src_f32 = 1;
  h.H = d->H; h.groups = lm.c.norm_groups; h.K = lm.Hp; h.eps = (float)lm.c.norm_eps; h.ldw = lm.Hp;
  h.W1 = d->head_w; h.n1 = d->lnf_w; h.N1 = d->V; h.out1 = d->logits;
  return launch_latent_in(st, h);
}

int forward_latent(rai_hip_decoder *d, int B, int S, bool advance_step, bool from_tokens) {
  hipStream_t st = stream_of(d->dev);
  if (!st) return RAI_ERR_HIP;
  LatentModel &lm = *d->latent;
  const int dt = d->cfg.dtype, Hp = lm.Hp;
  const int64_t M = (int64_t)B * S;
  RAI_TRY(ensure_derived(d, st));
  if (!from_tokens) RAI_TRY(decoder_embed(d, st, M));
  if (M == 1 && single_row_ok(d)) {
    RAI_TRY(single_row_layers(d, st));
    RAI_TRY(launch_token_choice(d, st, B, S, advance_step));
    d->ctx_len += S;
    return RAI_OK;
  }

  const bool frag = wants_fragments(d, M);
  if (frag || wants_fragments(d, B)) RAI_TRY(ensure_latent_fragments(d, st));
  const LatentLayer *pending = nullptr;   // the mixture whose outputs are not yet part of the stream
  for (int l = 0; l < d->L; ++l) {
    const LatentLayer &y = lm.layers[l];
    StreamNormArgs n = stream_norm_args(d, M);
    if (l == 0) {
      n.src = d->x; n.src_f32 = 0; n.src_ld = d->H;
      n.x = lm.xs;
    }
    add_pending(d, pending, &n);
    pending = nullptr;
    n.w1 = y.n1_w; n.h1 = lm.h1;
    if (y.n2_w) { n.w2 = y.n2_w; n.h2 = lm.h2; }
    RAI_TRY(launch_stream_norm(st, dt, n));

    LinearArgs a = latent_linear_args(d, lm.h1, Hp, M, y.Wd, y.ldn, Hp);
    a.out1 = lm.dn; a.ld1 = y.ldn;
    a.Wfrag = frag ? y.Wd_f : nullptr;
    RAI_TRY(decoder_linear(d, st, a));
    const bool absorb = S < kAbsorbRows;
    LatentNormArgs ln;
    memset(&ln, 0, sizeof(ln));
    ln.dn = lm.dn; ln.ldn = y.ldn;
    ln.q_rank = y.c.q_rank; ln.Qp = y.Qp; ln.kv_rank = y.c.kv_rank; ln.Rp = y.Rp;
    ln.q_w = y.q_w; ln.c_w = y.c_w;
    ln.cq = lm.cq; ln.cn = absorb ? nullptr : lm.cn; ln.cache = y.cache;
    ln.state = d->state;
    ln.B = B; ln.S = S; ln.Tmax = d->cfg.max_context;
    ln.eps = (float)lm.c.norm_eps;
    RAI_TRY(launch_latent_norm(st, dt, ln));
    LinearArgs q = latent_linear_args(d, lm.cq, y.Qp, M, y.Wuq, y.QD, y.Qp);
    q.out1 = lm.q; q.ld1 = y.QD;
    q.Wfrag = frag ? y.Wuq_f : nullptr;
    RAI_TRY(decoder_linear(d, st, q));
    RAI_TRY(absorb ? absorbed_attention(d, st, y, B, S) : expanded_attention(d, st, y, B, S));

    if (y.c.mlp_kind == RAI_MLP_DENSE) {
      LinearArgs g = latent_linear_args(d, lm.h2, Hp, M, y.Wgu, 2 * y.Fp, Hp);
      g.out1 = lm.cat + (size_t)y.QD * d->es; g.ld1 = y.QD + y.Fp;
      g.Wfrag = frag ? y.Wgu_f : nullptr;
      g.act = y.c.mlp_act; g.act_from = 0; g.glu = 1;
      RAI_TRY(decoder_linear(d, st, g));
    }
    RAI_TRY(residual_linear(d, st, lm.cat, y.QD + y.Fp, M, y.Wb, y.QD + y.Fp, frag ? y.Wb_f : nullptr));
    if (y.c.mlp_kind == RAI_MLP_MIXTURE) {
      RAI_TRY(mixture(d, st, y, M, &pending));
    }
  }

  if (d->want_hidden && pending) {   // every row of the finished stream is asked for
    StreamNormArgs n = stream_norm_args(d, M);
    add_pending(d, pending, &n);
    pending = nullptr;
    RAI_TRY(launch_stream_norm(st, dt, n));
  }
  StreamNormArgs n = stream_norm_args(d, B);
  add_pending(d, pending, &n);
  n.x = nullptr;
  n.first = S - 1; n.step = S;
  n.w1 = d->lnf_w; n.h1 = d->last;
  RAI_TRY(launch_stream_norm(st, dt, n));
  LinearArgs h = latent_linear_args(d, d->last, Hp, B, d->head_w, d->V, Hp);
  h.out1 = d->logits; h.ld1 = d->V;
  h.Wfrag = wants_fragments(d, B) ? d->head_f : nullptr;
  RAI_TRY(decoder_linear(d, st, h));
  RAI_TRY(launch_token_choice(d, st, B, S, advance_step));
  d->ctx_len += S;
  return RAI_OK;
}

int latent_head_rows(rai_hip_decoder *d, hipStream_t st, const int *rows_dev, int n_rows, char *logits) {
  LatentModel &lm = *d->latent;
  StreamNormArgs n = stream_norm_args(d, n_rows);
  n.row_map = rows_dev;
  n.w1 = d->lnf_w; n.h1 = lm.h1;
  RAI_TRY(launch_stream_norm(st, d->cfg.dtype, n));
  LinearArgs h = latent_linear_args(d, lm.h1, lm.Hp, n_rows, d->head_w, d->V, lm.Hp);
  h.out1 = logits; h.ld1 = d->V;
  return decoder_linear(d, st, h);
}

int latent_hidden_to_host(rai_hip_decoder *d, int64_t rows, float *out) {
  RAI_HIP_TRY(hipStreamSynchronize(stream_of(d->dev)));
  RAI_HIP_TRY(hipMemcpy2D(out, (size_t)d->H * 4, d->latent->xs, (size_t)d->latent->Hp * 4, (size_t)d->H * 4, (size_t)rows, hipMemcpyDeviceToHost));
  return RAI_OK;
}

static bool known_act(int act) {
  return act == RAI_UN_NEW_GELU || act == RAI_UN_GELU || act == RAI_UN_SILU || act == RAI_UN_RELU;
}

}  // namespace rai

extern "C" int rai_hip_decoder_create_latent(int dev, const rai_hip_latent_config *cfg, const rai_hip_latent_layer *layers,
                                             rai_hip_decoder **out) {
  RAI_REQUIRE(cfg && layers && out, RAI_ERR_BAD_ARG, "decoder_create_latent: null argument");
  RAI_REQUIRE(cfg->dtype == RAI_BF16 || cfg->dtype == RAI_F32, RAI_ERR_BAD_DTYPE, "decoder_create_latent: bf16 or f32");
  RAI_REQUIRE(cfg->vocab_size > 0 && cfg->width > 0 && cfg->num_layers > 0 && cfg->norm_groups > 0 && cfg->width % cfg->norm_groups == 0 &&
                  cfg->max_batch > 0 && cfg->max_context > 0,
              RAI_ERR_BAD_ARG, "decoder_create_latent: bad config");
  int ff = 1;
  for (int l = 0; l < cfg->num_layers; ++l) {
    const rai_hip_latent_layer &c = layers[l];
    RAI_REQUIRE(c.heads > 0 && c.qk_dim > 0 && c.v_dim > 0 && c.q_rank > 0 && c.kv_rank > 0 && c.window >= 0, RAI_ERR_BAD_ARG,
                "decoder_create_latent: bad attention sizes in layer %d", l);
    RAI_REQUIRE(c.mlp_kind == RAI_MLP_NONE || c.mlp_kind == RAI_MLP_DENSE || c.mlp_kind == RAI_MLP_MIXTURE, RAI_ERR_BAD_ARG,
                "decoder_create_latent: mlp kind %d in layer %d", c.mlp_kind, l);
    RAI_REQUIRE(c.mlp_kind == RAI_MLP_NONE || (c.intermediate > 0 && known_act(c.mlp_act)), RAI_ERR_BAD_ARG,
                "decoder_create_latent: bad MLP in layer %d", l);
    RAI_REQUIRE(c.mlp_kind != RAI_MLP_MIXTURE || (c.experts > 0 && c.experts <= 2048 && c.top > 0 && c.top <= c.experts), RAI_ERR_BAD_ARG,
                "decoder_create_latent: top %d of %d experts in layer %d", c.top, c.experts, l);
    if (c.intermediate > ff) ff = c.intermediate;
  }
  if (!ctx(dev)) return RAI_ERR_HIP;
  rai_hip_decoder_config base;
  memset(&base, 0, sizeof(base));
  base.arch = RAI_ARCH_LELITAR;
  base.dtype = cfg->dtype;
  base.vocab_size = cfg->vocab_size;
  base.hidden_size = cfg->width;
  base.intermediate_size = ff;
  base.num_hidden_layers = cfg->num_layers;
  base.num_attention_heads = base.num_key_value_heads = layers[0].heads;
  base.head_dim = layers[0].qk_dim;
  base.max_position_embeddings = cfg->max_context;   // positions enter nothing but the window
  base.max_batch = cfg->max_batch;
  base.max_context = cfg->max_context;
  base.norm_eps = cfg->norm_eps;
  rai_hip_decoder *d = new rai_hip_decoder();
  decoder_init_fields(d, dev, base);
  d->embed_scale = 1.0f;
  d->latent = new LatentModel();
  d->latent->c = *cfg;
  const int st = create_latent(d, *cfg, layers);
  if (st != RAI_OK) {
    rai_hip_decoder_destroy(d);
    return st;
  }
  *out = d;
  return RAI_OK;
}
