// Driver of the hybrid decoders (RAI_ARCH_BEZADRA): a parallel block with one layer norm over an f32 residual stream,
//   x <- x + (mixer(n(x)) + mlp(n(x))),
// the mixer attention or the gated delta rule, a run of layers looped with the same weights.
//
// A looped layer is run once per pass, and every run has a cache or state of its own (HybridRun).  Ahead of a pass,
// x <- Wx x + W0 x0 + step[t]; W0 x0 is the same for every pass and is formed once per call.
//
// Per layer run:
//   stream norm -> Wd . h -> [q | k | v | gate] or [q | k | v | beta | a1 | g1];  gate|up . h with the gated epilogue
//   attention:  rotation + cache append, flash or row attention with cap, sink and gate; one token: the decode kernel
//   delta rule: a2 . a1 -> decays, g2 . g1 -> output gate, then delta.hip
//   [o | down] as one contraction with the f32 residual epilogue
// One bf16 row (decode): norm + both products in one launch, the mixer, [o | down] in one launch.
#include <cmath>

#include "decoder.h"

namespace rai {

static int pad32(int n) { return (n + 31) / 32 * 32; }
static int pad_key(int n) { return n > 32 && n <= 64 ? 64 : n > 64 && n <= 128 ? 128 : n > 128 && n <= 256 ? 256 : pad32(n); }   // what the chunked form serves

// Tables are shared by the layers that turn alike.
static int rotary_for(rai_hip_decoder *d, const RotaryParams &r, const float **cos_t, const float **sin_t) {
  HybridModel &hm = *d->hybrid;
  for (const auto &t : hm.tables)
    if (same_rotary(t.first, r)) {
      *cos_t = t.second.first;
      *sin_t = t.second.second;
      return RAI_OK;
    }
  std::vector<float> cs, sn;
  rotary_tables(r, d->cfg.max_context, &cs, &sn);
  char *c = nullptr, *s = nullptr;
  RAI_TRY(dalloc(d, cs.size() * sizeof(float), &c));
  RAI_TRY(dalloc(d, sn.size() * sizeof(float), &s));
  if (!cs.empty()) {
    RAI_HIP_TRY(hipMemcpy(c, cs.data(), cs.size() * sizeof(float), hipMemcpyHostToDevice));
    RAI_HIP_TRY(hipMemcpy(s, sn.data(), sn.size() * sizeof(float), hipMemcpyHostToDevice));
  }
  hm.tables.push_back({r, {(const float *)c, (const float *)s}});
  *cos_t = (const float *)c;
  *sin_t = (const float *)s;
  return RAI_OK;
}

static int create_attention(rai_hip_decoder *d, HybridLayer &y, const std::string &mix) {
  const rai_hip_hybrid_layer &c = y.c;
  const size_t es = d->es;
  const int Hp = d->hybrid->Hp, KD = c.kv_heads * y.Dp;
  auto rows = [&](const char *name, int heads, int dim, int64_t first) {
    add_grouped_slot(d, mix + name, (int64_t)heads * dim, d->H, y.Wd + (size_t)first * Hp * es, Hp, dim, (int64_t)y.Dp * Hp, 0, 0);
  };
  rows("q", c.heads, c.qk_dim, 0);
  rows("k", c.kv_heads, c.qk_dim, y.QD);
  rows("v", c.kv_heads, c.v_dim, y.QD + KD);
  rows("g", c.heads, c.v_dim, y.QD + 2 * KD);
  RAI_TRY(zalloc(d, (size_t)c.heads * es, &y.sink));
  add_slot(d, mix + "sink", 1, c.heads, y.sink, c.heads);
  add_grouped_slot(d, mix + "o", d->H, (int64_t)c.heads * c.v_dim, y.Wb, y.QD + y.Fp, 0, 0, c.v_dim, y.Dp);
  return rotary_for(d, RotaryParams{c.rot_dims, c.rot_base, c.rot_factor, c.rot_low, c.rot_high, c.rot_original}, &y.cos_t, &y.sin_t);
}

static int create_delta(rai_hip_decoder *d, HybridLayer &y, const std::string &mix) {
  const rai_hip_hybrid_layer &c = y.c;
  const DeltaShape &z = y.delta;
  const size_t es = d->es;
  const int Hp = d->hybrid->Hp, kd = z.kv_heads * z.Dk;
  RAI_TRY(zalloc(d, (size_t)z.channels * z.taps * es, &y.conv));
  auto rows = [&](const char *name, int heads, int dim, int padded, int64_t first) {
    add_grouped_slot(d, mix + name, (int64_t)heads * dim, d->H, y.Wd + (size_t)first * Hp * es, Hp, dim, (int64_t)padded * Hp, 0, 0);
    add_grouped_slot(d, mix + name + ".conv", (int64_t)heads * dim, z.taps, y.conv + (size_t)first * z.taps * es, z.taps, dim,
                     (int64_t)padded * z.taps, 0, 0);
  };
  rows("q", z.kv_heads, z.dim, z.Dk, 0);
  rows("k", z.kv_heads, z.dim, z.Dk, kd);
  rows("v", z.heads, z.vdim, z.Vp, 2 * kd);
  add_slot(d, mix + "b", z.heads, d->H, y.Wd + (size_t)z.off_b * Hp * es, Hp);
  add_slot(d, mix + "a1", c.decay_rank, d->H, y.Wd + (size_t)z.off_a1 * Hp * es, Hp);
  add_slot(d, mix + "g1", c.gate_rank, d->H, y.Wd + (size_t)z.off_g1 * Hp * es, Hp);
  RAI_TRY(zalloc(d, (size_t)z.heads * es, &y.A_log));
  RAI_TRY(zalloc(d, (size_t)z.heads * z.Dk * es, &y.dt_bias));
  RAI_TRY(zalloc(d, (size_t)z.Vp * es, &y.norm_w));
  RAI_TRY(zalloc(d, (size_t)z.heads * z.Dk * y.a_rank * es, &y.a2));
  RAI_TRY(zalloc(d, (size_t)z.heads * z.Vp * y.g_rank * es, &y.g2));
  add_slot(d, mix + "A_log", 1, z.heads, y.A_log, z.heads);
  add_grouped_slot(d, mix + "dt_bias", 1, (int64_t)z.heads * z.dim, y.dt_bias, (int64_t)z.heads * z.Dk, 0, 0, z.dim, z.Dk);
  add_slot(d, mix + "norm", 1, z.vdim, y.norm_w, z.vdim);
  add_grouped_slot(d, mix + "a2", (int64_t)z.heads * z.dim, c.decay_rank, y.a2, y.a_rank, z.dim, (int64_t)z.Dk * y.a_rank, 0, 0);
  add_grouped_slot(d, mix + "g2", (int64_t)z.heads * z.vdim, c.gate_rank, y.g2, y.g_rank, z.vdim, (int64_t)z.Vp * y.g_rank, 0, 0);
  add_grouped_slot(d, mix + "o", d->H, (int64_t)z.heads * z.vdim, y.Wb, y.QD + y.Fp, 0, 0, z.vdim, z.Vp);
  return RAI_OK;
}

static int create_layer(rai_hip_decoder *d, int l, const rai_hip_hybrid_layer &c) {
  HybridModel &hm = *d->hybrid;
  HybridLayer y;
  memset(&y, 0, sizeof(y));
  y.c = c;
  const size_t es = d->es;
  const int H = d->H, Hp = hm.Hp;
  y.Fp = c.mlp_kind == RAI_MLP_DENSE ? pad64(c.intermediate) : 0;
  if (c.mixer == RAI_MIXER_ATTENTION) {
    y.Dp = pad_head(c.qk_dim > c.v_dim ? c.qk_dim : c.v_dim);
    y.QD = c.heads * y.Dp;
    y.ldn = 2 * y.QD + 2 * c.kv_heads * y.Dp;
  } else {
    DeltaShape &z = y.delta;
    z.heads = c.heads; z.kv_heads = c.kv_heads; z.dim = c.qk_dim; z.vdim = c.v_dim; z.taps = c.conv_taps;
    z.Dk = pad_key(c.qk_dim); z.Vp = pad32(c.v_dim);
    y.a_rank = pad64(c.decay_rank); y.g_rank = pad64(c.gate_rank);
    z.channels = 2 * z.kv_heads * z.Dk + z.heads * z.Vp;
    z.off_b = pad64(z.channels);
    z.off_a1 = z.off_b + pad64(z.heads);
    z.off_g1 = z.off_a1 + y.a_rank;
    y.ldn = z.off_g1 + y.g_rank;
    z.ldn = y.ldn;
    y.QD = pad64(z.heads * z.Vp);
  }
  RAI_TRY(zalloc(d, (size_t)H * es, &y.n1_w));
  RAI_TRY(zalloc(d, (size_t)y.ldn * Hp * es, &y.Wd));
  RAI_TRY(zalloc(d, (size_t)Hp * (y.QD + y.Fp) * es, &y.Wb));
  const std::string p = "l" + std::to_string(l) + ".";
  add_slot(d, p + "norm1", 1, H, y.n1_w, H);
  RAI_TRY(c.mixer == RAI_MIXER_ATTENTION ? create_attention(d, y, p + "mix.") : create_delta(d, y, p + "mix."));
  if (y.Fp) {
    RAI_TRY(zalloc(d, (size_t)2 * y.Fp * Hp * es, &y.Wgu));
    add_slot(d, p + "mlp.gate", c.intermediate, H, y.Wgu, 2 * (int64_t)Hp);
    add_slot(d, p + "mlp.up", c.intermediate, H, y.Wgu + (size_t)Hp * es, 2 * (int64_t)Hp);
    add_slot(d, p + "mlp.down", H, c.intermediate, y.Wb + (size_t)y.QD * es, y.QD + y.Fp);
  }
  hm.layers.push_back(y);
  return RAI_OK;
}

static int create_run(rai_hip_decoder *d, int layer, int pass) {
  HybridModel &hm = *d->hybrid;
  const HybridLayer &y = hm.layers[layer];
  HybridRun r;
  memset(&r, 0, sizeof(r));
  r.layer = layer;
  r.pass = pass;
  const size_t B = d->cfg.max_batch;
  if (y.c.mixer == RAI_MIXER_ATTENTION) {
    const size_t bytes = B * y.c.kv_heads * d->cfg.max_context * y.Dp * d->es;
    RAI_TRY(zalloc(d, bytes, &r.kcache));
    RAI_TRY(zalloc(d, bytes, &r.vcache));
  } else {
    char *tmp = nullptr;
    RAI_TRY(zalloc(d, B * y.delta.taps * y.delta.channels * d->es, &r.ring));
    RAI_TRY(zalloc(d, B * y.delta.heads * y.delta.Dk * y.delta.Vp * sizeof(float), &tmp));
    r.carried = (float *)tmp;
  }
  hm.runs.push_back(r);
  return RAI_OK;
}

static int create_hybrid(rai_hip_decoder *d, const rai_hip_hybrid_config &cfg, const rai_hip_hybrid_layer *layers) {
  HybridModel &hm = *d->hybrid;
  const size_t es = d->es;
  const int H = d->H, Hp = hm.Hp = pad64(H), V = d->V;
  RAI_TRY(decoder_alloc_common(d));
  RAI_TRY(zalloc(d, (size_t)V * H * es, &d->embed));
  add_slot(d, "embed", V, H, d->embed, H);
  d->head_w = d->embed;
  if (H != Hp) RAI_TRY(zalloc(d, (size_t)V * Hp * es, &d->head_w));
  d->head_b = nullptr;
  if (cfg.loop_times > 0) {
    const size_t half = (size_t)Hp * Hp;
    char *w = nullptr;
    RAI_TRY(zalloc(d, 2 * half * es, &w));
    hm.Wx = w;
    hm.W0 = w + half * es;
    RAI_TRY(zalloc(d, (size_t)cfg.loop_times * Hp * es, &hm.step));
    add_grouped_slot(d, "loop.in", H, 2 * (int64_t)H, hm.Wx, Hp, 0, 0, H, (int64_t)half);
    add_slot(d, "loop.step", cfg.loop_times, H, hm.step, Hp);
  }
  for (int l = 0; l < cfg.num_layers; ++l) RAI_TRY(create_layer(d, l, layers[l]));
  RAI_TRY(zalloc(d, (size_t)H * es, &d->lnf_w));
  add_slot(d, "final.norm", 1, H, d->lnf_w, H);
  const int start = cfg.loop_times > 0 ? cfg.loop_start : cfg.num_layers, stop = cfg.loop_times > 0 ? cfg.loop_stop : cfg.num_layers;
  for (int l = 0; l < start; ++l) RAI_TRY(create_run(d, l, -1));
  for (int t = 0; t < cfg.loop_times; ++t)
    for (int l = start; l < stop; ++l) RAI_TRY(create_run(d, l, l == start ? t : -1));
  for (int l = stop; l < cfg.num_layers; ++l) RAI_TRY(create_run(d, l, -1));

  // activations, sized for the widest layer
  const int64_t rows = d->max_rows;
  int ldn = 0, KB = 0;
  size_t decay = 0, qk = 0, kvh = 0, val = 0, beta = 0, ws = 0, counters = 0, chunk = 0;
  for (const HybridLayer &y : hm.layers) {
    ldn = std::max(ldn, y.ldn);
    KB = std::max(KB, y.QD + y.Fp);
    if (y.c.mixer == RAI_MIXER_ATTENTION) {
      ws = std::max(ws, attention_decode_ws_bytes(cfg.max_batch, y.c.heads, y.Dp));
      counters = std::max(counters, attention_decode_counter_bytes(cfg.max_batch, y.c.heads));
    } else {
      const DeltaShape &z = y.delta;
      decay = std::max(decay, (size_t)z.heads * z.Dk);
      qk = std::max(qk, (size_t)z.kv_heads * z.Dk);
      kvh = std::max(kvh, (size_t)z.kv_heads);
      val = std::max(val, (size_t)z.heads * z.Vp);
      if (delta_chunk_serves(cfg.dtype, z)) chunk = std::max(chunk, delta_chunk_ws_bytes(z, cfg.max_batch, rows));
      beta = std::max(beta, (size_t)z.heads);
    }
  }
  auto floats = [&](size_t per_row, float **out) -> int {
    char *tmp = nullptr;
    RAI_TRY(zalloc(d, rows * per_row * sizeof(float), &tmp));
    *out = (float *)tmp;
    return RAI_OK;
  };
  RAI_TRY(zalloc(d, rows * H * es, &d->x));
  RAI_TRY(floats(Hp, &hm.xs));
  char *tmp = nullptr;
  RAI_TRY(zalloc(d, Hp * sizeof(float), &tmp));   // only the single-row step swaps
  hm.xs2 = (float *)tmp;
  if (cfg.loop_times > 0) RAI_TRY(floats(Hp, &hm.x0w));
  RAI_TRY(zalloc(d, rows * Hp * es, &hm.h1));
  RAI_TRY(zalloc(d, rows * ldn * es, &hm.dn));
  RAI_TRY(zalloc(d, rows * KB * es, &hm.cat));
  RAI_TRY(zalloc(d, (size_t)cfg.max_batch * Hp * es, &d->last));
  if (val) {
    RAI_TRY(floats(decay, &hm.decay));
    RAI_TRY(zalloc(d, rows * qk * es, &hm.dq));
    RAI_TRY(zalloc(d, rows * qk * es, &hm.dk));
    RAI_TRY(floats(kvh, &hm.qn));
    RAI_TRY(floats(kvh, &hm.kn));
    RAI_TRY(zalloc(d, rows * val * es, &hm.dv));
    if (chunk) RAI_TRY(zalloc(d, chunk, &hm.chunk_ws));
    RAI_TRY(floats(beta, &hm.beta));
    RAI_TRY(zalloc(d, (rows + 1) * val * sizeof(float), &tmp));
    hm.o = (float *)tmp;
    RAI_TRY(zalloc(d, rows * val * es, &hm.gate));
  }
  if (ws) {
    RAI_TRY(zalloc(d, ws, &hm.attn_ws));
    RAI_TRY(zalloc(d, counters, &tmp));
    hm.attn_counters = (int *)tmp;
  }
  hm.stream = hm.xs;
  return RAI_OK;
}

// ------------------------------------------------------------------ forward
static int ensure_derived(rai_hip_decoder *d, hipStream_t st) {
  HybridModel &hm = *d->hybrid;
  if (hm.derived_ready) return RAI_OK;
  if (d->head_w != d->embed)
    RAI_HIP_TRY(hipMemcpy2DAsync(d->head_w, (size_t)hm.Hp * d->es, d->embed, (size_t)d->H * d->es, (size_t)d->H * d->es, d->V, hipMemcpyDeviceToDevice, st));
  hm.derived_ready = true;
  return RAI_OK;
}

static int ensure_hybrid_fragments(rai_hip_decoder *d, hipStream_t st) {
  HybridModel &hm = *d->hybrid;
  if (d->frag_ready) return RAI_OK;
  for (HybridLayer &y : hm.layers) {
    const int KB = y.QD + y.Fp;
    RAI_TRY(decoder_fragments(d, st, y.Wd, hm.Hp, y.ldn, hm.Hp, &y.Wd_f));
    RAI_TRY(decoder_fragments(d, st, y.Wgu, hm.Hp, 2 * y.Fp, hm.Hp, &y.Wgu_f));
    RAI_TRY(decoder_fragments(d, st, y.Wb, KB, hm.Hp, KB, &y.Wb_f));
    RAI_TRY(decoder_fragments(d, st, y.a2, y.a_rank, y.delta.heads * y.delta.Dk, y.a_rank, &y.a2_f));
    RAI_TRY(decoder_fragments(d, st, y.g2, y.g_rank, y.delta.heads * y.delta.Vp, y.g_rank, &y.g2_f));
  }
  RAI_TRY(decoder_fragments(d, st, hm.Wx, hm.Hp, hm.Hp, hm.Hp, &hm.Wx_f));
  RAI_TRY(decoder_fragments(d, st, hm.W0, hm.Hp, hm.Hp, hm.Hp, &hm.W0_f));
  RAI_TRY(decoder_fragments(d, st, d->head_w, hm.Hp, d->V, hm.Hp, &d->head_f));
  d->frag_ready = true;
  return RAI_OK;
}

static LinearArgs hybrid_linear_args(rai_hip_decoder *d, const void *A, int64_t lda, int64_t M, const char *W, int N, int K, const char *Wfrag) {
  LinearArgs a = linear_args_default();
  a.A = A; a.lda = lda;
  a.W = W; a.ldw = K;
  a.M = (int)M; a.N = N; a.K = K; a.n_split = N;
  a.Wfrag = wants_fragments(d, M) ? Wfrag : nullptr;
  a.splitk_ws = d->splitk_ws; a.splitk_ws_bytes = d->splitk_ws_bytes;
  return a;
}
// out (f32) = A W^T [+ bias] [+ residual (f32)]
static int f32_linear(rai_hip_decoder *d, hipStream_t st, LinearArgs a, float *out, int64_t ldo, const float *residual, const void *bias) {
  a.out1 = out; a.ld1 = ldo;
  a.residual = residual; a.ldr = ldo;
  a.bias = bias;
  a.f32_out = 1; a.out_scale = 1.f;
  return decoder_linear(d, st, a);
}

static StreamNormArgs hybrid_norm_args(rai_hip_decoder *d, int64_t rows, int kind) {
  HybridModel &hm = *d->hybrid;
  StreamNormArgs n;
  memset(&n, 0, sizeof(n));
  n.src = hm.xs; n.src_f32 = 1; n.src_ld = hm.Hp;
  n.x_ld = hm.Hp; n.h_ld = hm.Hp;
  n.width = d->H; n.groups = 1; n.eps = (float)hm.c.norm_eps;
  n.rows = rows; n.first = 0; n.step = 1;
  n.kind = kind;
  return n;
}
static void from_embedding(rai_hip_decoder *d, StreamNormArgs *n) {
  n->src = d->x; n->src_f32 = 0; n->src_ld = d->H;
  n->src_scale = (float)d->hybrid->c.embed_scale;
}

static AttnDecodeArgs decode_attention_args(rai_hip_decoder *d, const HybridLayer &y, const HybridRun &r, int B) {
  HybridModel &hm = *d->hybrid;
  const size_t es = d->es;
  const int KD = y.c.kv_heads * y.Dp;
  AttnDecodeArgs t;
  memset(&t, 0, sizeof(t));
  t.qkv = hm.dn; t.k_new = hm.dn + (size_t)y.QD * es; t.v_new = hm.dn + (size_t)(y.QD + KD) * es;
  t.q_row_stride = t.k_row_stride = t.v_row_stride = y.ldn;
  t.kcache = r.kcache; t.vcache = r.vcache;
  t.out = hm.cat; t.out_row_stride = y.QD + y.Fp;
  t.cos_t = y.cos_t; t.sin_t = y.sin_t; t.tab_f32 = 1; t.rot = y.c.rot_dims;
  t.pos_dev = &d->state->pos;
  t.B = B; t.Hq = y.c.heads; t.Hkv = y.c.kv_heads; t.D = y.Dp; t.Tmax = d->cfg.max_context;
  t.scale = (float)y.c.attn_scale; t.softcap = (float)y.c.softcap; t.f32_scores = 1;
  t.sink = y.sink;
  t.gate = hm.dn + (size_t)(y.QD + 2 * KD) * es; t.gate_row_stride = y.ldn;
  t.dtype = d->cfg.dtype;
  t.ws = (float *)hm.attn_ws; t.counters = hm.attn_counters;
  return t;
}
static bool decode_attention_serves(const rai_hip_decoder *d, const HybridLayer &y) { return (size_t)y.Dp * d->es <= 1024; }

static int attention_mixer(rai_hip_decoder *d, hipStream_t st, const HybridLayer &y, const HybridRun &r, int B, int S) {
  HybridModel &hm = *d->hybrid;
  if (S == 1 && decode_attention_serves(d, y)) return launch_attention_decode(st, decode_attention_args(d, y, r, B));
  const size_t es = d->es;
  const int64_t Tmax = d->cfg.max_context;
  RotaryAppendArgs ra;
  memset(&ra, 0, sizeof(ra));
  ra.rows = hm.dn; ra.ld = y.ldn; ra.kcache = r.kcache; ra.vcache = r.vcache;
  ra.cos_t = y.cos_t; ra.sin_t = y.sin_t; ra.state = d->state;
  ra.B = B; ra.S = S; ra.heads = y.c.heads; ra.kv_heads = y.c.kv_heads; ra.D = y.Dp; ra.rot = y.c.rot_dims; ra.Tmax = (int)Tmax;
  RAI_TRY(launch_rotary_append(st, d->cfg.dtype, ra));
  AttnArgs t;
  memset(&t, 0, sizeof(t));
  t.q = hm.dn; t.k = r.kcache; t.v = r.vcache;
  t.out = hm.cat; t.out_row_stride = y.QD + y.Fp;
  t.qs[0] = (int64_t)S * y.ldn; t.qs[1] = y.Dp; t.qs[2] = y.ldn;
  t.ks[0] = t.vs[0] = y.c.kv_heads * Tmax * y.Dp; t.ks[1] = t.vs[1] = Tmax * y.Dp; t.ks[2] = t.vs[2] = y.Dp;
  t.B = B; t.Hq = y.c.heads; t.Hkv = y.c.kv_heads; t.S = S; t.T = d->ctx_len + S; t.D = y.Dp;
  if (S == 1) {   // a step that is replayed from a graph: the length is the device's
    t.T = (int)Tmax;
    t.t_dev = &d->state->pos; t.t_add = 1;
  }
  t.scale = (float)y.c.attn_scale; t.softcap = (float)y.c.softcap; t.sink = y.sink;
  t.causal = 1; t.f32_scores = 1; t.dtype = d->cfg.dtype;
  t.gate = hm.dn + (size_t)(y.QD + 2 * y.c.kv_heads * y.Dp) * es; t.gate_row_stride = y.ldn;
  return launch_attention(st, t);
}

static DeltaArgs delta_args(rai_hip_decoder *d, const HybridLayer &y, const HybridRun &r, int B, int S) {
  HybridModel &hm = *d->hybrid;
  DeltaArgs a;
  memset(&a, 0, sizeof(a));
  a.s = y.delta; a.B = B; a.S = S; a.state = d->state;
  a.dn = hm.dn; a.conv = y.conv; a.ring = r.ring; a.carried = r.carried;
  a.A_log = y.A_log; a.dt_bias = y.dt_bias;
  a.decay = hm.decay; a.q = hm.dq; a.k = hm.dk; a.qn = hm.qn; a.kn = hm.kn; a.v = hm.dv; a.beta = hm.beta; a.o = hm.o;
  a.norm_w = y.norm_w; a.eps = (float)hm.c.norm_eps;
  a.gate = hm.gate;
  a.chunk_ws = hm.chunk_ws;
  a.out = hm.cat; a.ldo = y.QD + y.Fp;
  return a;
}

static int delta_mixer(rai_hip_decoder *d, hipStream_t st, const HybridLayer &y, const HybridRun &r, int B, int S) {
  HybridModel &hm = *d->hybrid;
  const DeltaShape &z = y.delta;
  const int64_t M = (int64_t)B * S;
  RAI_TRY(f32_linear(d, st, hybrid_linear_args(d, hm.dn + (size_t)z.off_a1 * d->es, y.ldn, M, y.a2, z.heads * z.Dk, y.a_rank, y.a2_f), hm.decay,
                     (int64_t)z.heads * z.Dk, nullptr, nullptr));
  LinearArgs g = hybrid_linear_args(d, hm.dn + (size_t)z.off_g1 * d->es, y.ldn, M, y.g2, z.heads * z.Vp, y.g_rank, y.g2_f);
  g.out1 = hm.gate; g.ld1 = (int64_t)z.heads * z.Vp;
  RAI_TRY(decoder_linear(d, st, g));
  const DeltaArgs a = delta_args(d, y, r, B, S);
  return S == 1 && delta_step_serves(z) ? launch_delta_step(st, d->cfg.dtype, a) : launch_delta_tokens(st, d->cfg.dtype, a);
}

// One bf16 row: norm and both products of it in one launch, the mixer, [o | down] with the residual in one launch.
static bool single_row_ok(const rai_hip_decoder *d) {
  int64_t cols = 0;
  for (const HybridLayer &y : d->hybrid->layers) {
    cols = std::max<int64_t>(cols, y.QD + y.Fp);
    if (y.c.mixer == RAI_MIXER_ATTENTION ? !decode_attention_serves(d, y) : !delta_step_serves(y.delta)) return false;
  }
  return d->cfg.dtype == RAI_BF16 && latent_single_row_serves(d->H, 1, 0, 0, cols);
}

static LatentInArgs row_in_args(rai_hip_decoder *d, const float *src, int kind) {   // src null: the embedding row
  HybridModel &hm = *d->hybrid;
  LatentInArgs in;
  memset(&in, 0, sizeof(in));
  in.src = src ? (const void *)src : (const void *)d->x;
  in.src_f32 = src != nullptr;
  in.src_scale = src ? 0.f : (float)hm.c.embed_scale;
  in.H = d->H; in.groups = 1; in.K = hm.Hp; in.eps = (float)hm.c.norm_eps; in.ldw = hm.Hp;
  in.kind = kind;
  return in;
}

static int single_row_runs(rai_hip_decoder *d, hipStream_t st) {
  HybridModel &hm = *d->hybrid;
  const size_t es = d->es;
  float *cur = nullptr, *buf[2] = {hm.xs, hm.xs2};   // cur null: the stream is still the embedding row
  if (hm.c.loop_times > 0) {
    LatentInArgs in = row_in_args(d, nullptr, kStreamCopy);
    in.W2 = hm.W0; in.N2 = hm.Hp; in.out2 = hm.x0w;
    RAI_TRY(launch_latent_in(st, in));
  }
  for (const HybridRun &r : hm.runs) {
    const HybridLayer &y = hm.layers[r.layer];
    if (r.pass >= 0) {
      float *next = cur == buf[0] ? buf[1] : buf[0];
      LatentInArgs in = row_in_args(d, cur, kStreamCopy);
      in.W2 = hm.Wx; in.N2 = hm.Hp; in.out2 = next;
      in.add2 = hm.x0w; in.bias2 = hm.step + (size_t)r.pass * hm.Hp * es;
      RAI_TRY(launch_latent_in(st, in));
      cur = next;
    }
    LatentInArgs in = row_in_args(d, cur, kStreamLayerNorm);
    in.W1 = y.Wd; in.n1 = y.n1_w; in.N1 = y.ldn; in.out1 = hm.dn;
    in.n2 = y.n1_w;
    if (y.Fp) {
      in.W2 = y.Wgu; in.N2 = 2 * y.Fp; in.gated2 = 1; in.out2 = hm.cat + (size_t)y.QD * es;
      in.act = kActClampedGlu; in.act_limit = (float)y.c.mlp_limit; in.act_alpha = (float)y.c.mlp_alpha;
    }
    RAI_TRY(launch_latent_in(st, in));
    if (y.c.mixer == RAI_MIXER_ATTENTION) {
      RAI_TRY(launch_attention_decode(st, decode_attention_args(d, y, r, 1)));
    } else {
      DeltaArgs a = delta_args(d, y, r, 1, 1);
      a.a2 = y.a2; a.g2 = y.g2; a.a_rank = y.a_rank; a.g_rank = y.g_rank;
      RAI_TRY(launch_delta_step(st, d->cfg.dtype, a));
    }
    LatentDownArgs dn;
    memset(&dn, 0, sizeof(dn));
    dn.x0 = hm.cat; dn.W0 = y.Wb; dn.K0 = y.QD + y.Fp;
    dn.res = cur ? (const void *)cur : (const void *)d->x; dn.res_f32 = cur != nullptr;
    dn.res_scale = cur ? 0.f : (float)hm.c.embed_scale;
    dn.H = d->H; dn.N = hm.Hp; dn.rows = 1; dn.mult = 1.f;
    if (!cur) cur = buf[0];
    dn.out = cur;
    RAI_TRY(launch_latent_down(st, dn));
  }
  hm.stream = cur;
  LatentInArgs h = row_in_args(d, cur, kStreamLayerNorm);
  h.h_scale = (float)hm.c.logit_scale;
  h.W1 = d->head_w; h.n1 = d->lnf_w; h.N1 = d->V; h.out1 = d->logits;
  return launch_latent_in(st, h);
}

// Logits of n rows of the stream: first, first + step, ... or row_map.
static int head(rai_hip_decoder *d, hipStream_t st, int n_rows, int64_t first, int64_t step, const int *row_map, void *normed, char *logits) {
  HybridModel &hm = *d->hybrid;
  StreamNormArgs n = hybrid_norm_args(d, n_rows, kStreamLayerNorm);
  n.src = hm.stream;
  n.first = first; n.step = step; n.row_map = row_map;
  n.h_scale = (float)hm.c.logit_scale;
  n.w1 = d->lnf_w; n.h1 = normed;
  RAI_TRY(launch_stream_norm(st, d->cfg.dtype, n));
  LinearArgs h = hybrid_linear_args(d, normed, hm.Hp, n_rows, d->head_w, d->V, hm.Hp, d->frag_ready ? d->head_f : nullptr);
  h.out1 = logits; h.ld1 = d->V;
  return decoder_linear(d, st, h);
}

int forward_hybrid(rai_hip_decoder *d, int B, int S, bool advance_step, bool from_tokens) {
  hipStream_t st = stream_of(d->dev);
  if (!st) return RAI_ERR_HIP;
  HybridModel &hm = *d->hybrid;
  const int dt = d->cfg.dtype, Hp = hm.Hp;
  const int64_t M = (int64_t)B * S;
  RAI_TRY(ensure_derived(d, st));
  if (!from_tokens) RAI_TRY(decoder_embed(d, st, M));
  if (M == 1 && single_row_ok(d)) {
    RAI_TRY(single_row_runs(d, st));
    RAI_TRY(launch_token_choice(d, st, B, S, advance_step));
    d->ctx_len += S;
    return RAI_OK;
  }
  if (wants_fragments(d, M) || wants_fragments(d, B)) RAI_TRY(ensure_hybrid_fragments(d, st));
  hm.stream = hm.xs;
  bool embedding = true;   // the stream is still the embedding output, in d->x
  if (hm.c.loop_times > 0) {
    StreamNormArgs n = hybrid_norm_args(d, M, kStreamCopy);
    from_embedding(d, &n);
    n.h1 = hm.h1;
    RAI_TRY(launch_stream_norm(st, dt, n));
    RAI_TRY(f32_linear(d, st, hybrid_linear_args(d, hm.h1, Hp, M, hm.W0, Hp, Hp, hm.W0_f), hm.x0w, Hp, nullptr, nullptr));
  }
  for (const HybridRun &r : hm.runs) {
    const HybridLayer &y = hm.layers[r.layer];
    if (r.pass >= 0) {
      StreamNormArgs n = hybrid_norm_args(d, M, kStreamCopy);
      if (embedding) from_embedding(d, &n);
      n.h1 = hm.h1;
      RAI_TRY(launch_stream_norm(st, dt, n));
      RAI_TRY(f32_linear(d, st, hybrid_linear_args(d, hm.h1, Hp, M, hm.Wx, Hp, Hp, hm.Wx_f), hm.xs, Hp, hm.x0w, hm.step + (size_t)r.pass * Hp * d->es));
      embedding = false;
    }
    StreamNormArgs n = hybrid_norm_args(d, M, kStreamLayerNorm);
    if (embedding) {
      from_embedding(d, &n);
      n.x = hm.xs;
      embedding = false;
    }
    n.w1 = y.n1_w; n.h1 = hm.h1;
    RAI_TRY(launch_stream_norm(st, dt, n));
    LinearArgs a = hybrid_linear_args(d, hm.h1, Hp, M, y.Wd, y.ldn, Hp, y.Wd_f);
    a.out1 = hm.dn; a.ld1 = y.ldn;
    RAI_TRY(decoder_linear(d, st, a));
    const int KB = y.QD + y.Fp;
    if (y.Fp) {
      LinearArgs g = hybrid_linear_args(d, hm.h1, Hp, M, y.Wgu, 2 * y.Fp, Hp, y.Wgu_f);
      g.out1 = hm.cat + (size_t)y.QD * d->es; g.ld1 = KB;
      g.act = kActClampedGlu; g.act_from = 0; g.glu = 1;
      g.act_limit = (float)y.c.mlp_limit; g.act_alpha = (float)y.c.mlp_alpha;
      RAI_TRY(decoder_linear(d, st, g));
    }
    RAI_TRY(y.c.mixer == RAI_MIXER_ATTENTION ? attention_mixer(d, st, y, r, B, S) : delta_mixer(d, st, y, r, B, S));
    LinearArgs o = hybrid_linear_args(d, hm.cat, KB, M, y.Wb, Hp, KB, y.Wb_f);
    RAI_TRY(f32_linear(d, st, o, hm.xs, Hp, hm.xs, nullptr));
  }
  RAI_TRY(head(d, st, B, S - 1, S, nullptr, d->last, d->logits));
  RAI_TRY(launch_token_choice(d, st, B, S, advance_step));
  d->ctx_len += S;
  return RAI_OK;
}

int hybrid_head_rows(rai_hip_decoder *d, hipStream_t st, const int *rows_dev, int n_rows, char *logits) {
  return head(d, st, n_rows, 0, 1, rows_dev, d->hybrid->h1, logits);
}

int hybrid_hidden_to_host(rai_hip_decoder *d, int64_t rows, float *out) {
  RAI_HIP_TRY(hipStreamSynchronize(stream_of(d->dev)));
  RAI_HIP_TRY(hipMemcpy2D(out, (size_t)d->H * 4, d->hybrid->stream, (size_t)d->hybrid->Hp * 4, (size_t)d->H * 4, (size_t)rows, hipMemcpyDeviceToHost));
  return RAI_OK;
}

}  // namespace rai

extern "C" int rai_hip_decoder_create_hybrid(int dev, const rai_hip_hybrid_config *cfg, const rai_hip_hybrid_layer *layers, rai_hip_decoder **out) {
  RAI_REQUIRE(cfg && layers && out, RAI_ERR_BAD_ARG, "decoder_create_hybrid: null argument");
  RAI_REQUIRE(cfg->dtype == RAI_BF16 || cfg->dtype == RAI_F32, RAI_ERR_BAD_DTYPE, "decoder_create_hybrid: bf16 or f32");
  RAI_REQUIRE(cfg->vocab_size > 0 && cfg->width > 0 && cfg->num_layers > 0 && cfg->max_batch > 0 && cfg->max_context > 0, RAI_ERR_BAD_ARG,
              "decoder_create_hybrid: bad config");
  RAI_REQUIRE(cfg->loop_times >= 0 && (cfg->loop_times == 0 || (cfg->loop_start >= 0 && cfg->loop_start < cfg->loop_stop && cfg->loop_stop <= cfg->num_layers)),
              RAI_ERR_BAD_ARG, "decoder_create_hybrid: loop over layers %d .. %d of %d", cfg->loop_start, cfg->loop_stop, cfg->num_layers);
  int ff = 1;
  for (int l = 0; l < cfg->num_layers; ++l) {
    const rai_hip_hybrid_layer &c = layers[l];
    RAI_REQUIRE(c.heads > 0 && c.kv_heads > 0 && c.heads % c.kv_heads == 0 && c.qk_dim > 0 && c.v_dim > 0, RAI_ERR_BAD_ARG,
                "decoder_create_hybrid: %d / %d heads of %d / %d in layer %d", c.heads, c.kv_heads, c.qk_dim, c.v_dim, l);
    RAI_REQUIRE(c.mixer == RAI_MIXER_ATTENTION || c.mixer == RAI_MIXER_CHANNEL_DELTA, RAI_ERR_BAD_ARG, "decoder_create_hybrid: mixer %d in layer %d", c.mixer, l);
    if (c.mixer == RAI_MIXER_ATTENTION)
      RAI_REQUIRE(c.rot_dims >= 0 && c.rot_dims % 2 == 0 && c.rot_dims <= c.qk_dim && (!c.rot_dims || c.rot_base > 0) && c.softcap >= 0 &&
                      (c.rot_factor <= 0 || (c.rot_low > 0 && c.rot_high > c.rot_low && c.rot_original > 0)),
                  RAI_ERR_BAD_ARG, "decoder_create_hybrid: bad rotary positions or cap in layer %d", l);
    else
      RAI_REQUIRE(c.conv_taps > 0 && c.decay_rank > 0 && c.gate_rank > 0 && c.qk_dim <= kDeltaMaxHead && c.v_dim <= kDeltaMaxHead, RAI_ERR_BAD_ARG,
                  "decoder_create_hybrid: delta rule with %d taps, ranks %d and %d, heads of %d x %d in layer %d", c.conv_taps, c.decay_rank, c.gate_rank,
                  c.qk_dim, c.v_dim, l);
    RAI_REQUIRE(c.mlp_kind == RAI_MLP_NONE || (c.mlp_kind == RAI_MLP_DENSE && c.intermediate > 0), RAI_ERR_BAD_ARG, "decoder_create_hybrid: bad MLP in layer %d", l);
    if (c.intermediate > ff) ff = c.intermediate;
  }
  if (!ctx(dev)) return RAI_ERR_HIP;
  rai_hip_decoder_config base;
  memset(&base, 0, sizeof(base));
  base.arch = RAI_ARCH_BEZADRA;
  base.dtype = cfg->dtype;
  base.vocab_size = cfg->vocab_size;
  base.hidden_size = cfg->width;
  base.intermediate_size = ff;
  base.num_hidden_layers = cfg->num_layers;
  base.num_attention_heads = layers[0].heads;
  base.num_key_value_heads = layers[0].kv_heads;
  base.head_dim = layers[0].qk_dim;
  base.max_position_embeddings = cfg->max_context;
  base.max_batch = cfg->max_batch;
  base.max_context = cfg->max_context;
  base.norm_eps = cfg->norm_eps;
  rai_hip_decoder *d = new rai_hip_decoder();
  decoder_init_fields(d, dev, base);
  d->embed_scale = 1.0f;   // applied in f32 where the rows are read
  d->hybrid = new HybridModel();
  d->hybrid->c = *cfg;
  const int st = create_hybrid(d, *cfg, layers);
  if (st != RAI_OK) {
    rai_hip_decoder_destroy(d);
    return st;
  }
  *out = d;
  return RAI_OK;
}
