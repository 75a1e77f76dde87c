// The decoder object behind rai_hip_decoder_*, shared by the drivers of the model families (decoder.hip: Phi-2 and the
// sequential Qwen2 / Gemma / Phi-3 block; decoder_latent.hip: latent attention with a parallel MLP or mixture;
// decoder_hybrid.hip: attention and gated delta rule layers, some of them looped).
#pragma once
#include <map>
#include <string>
#include <vector>

#include "attention.h"
#include "decode_chain.h"
#include "decode_mega.h"
#include "delta.h"
#include "gemm.h"
#include "latent.h"
#include "rotary.h"

namespace rai {

struct ParamSlot {
  std::string name;
  int64_t rows, cols;       // logical [rows, cols] (1-D params: rows = 1)
  char *dst;                // device address of element [0, 0]
  int64_t pitch;            // elements between consecutive rows at dst
  bool loaded;
  // a parameter whose last rows2 rows go elsewhere (same pitch): Phi-3's gate_up_proj, whose gate rows and
  // up rows interleave in the packed matrix
  int64_t rows2;
  char *dst2;
  // Padded heads: the rows (columns) come in groups of row_group (col_group), each group starting row_stride
  // (col_stride) elements behind the one before; 0: no groups.
  int64_t row_group, row_stride, col_group, col_stride;
};

struct Layer {
  // Phi-2 (parallel block)
  char *Wa, *ba, *Wb, *bd, *bf, *ln_w, *ln_b;
  // Qwen2 / Gemma (sequential block): Wqkv [QD+2KD, H] (+bqkv), Wo [H, QD] (+bo),
  // Wgu [2I, H] with gate/up rows interleaved, Wdown [H, I], two RMSNorm weights
  char *Wqkv, *bqkv, *Wo, *bo, *Wgu, *Wdown, *n1_w, *n2_w;
  // second copies in MFMA-fragment order for the batched-decode streaming kernel (built on first use)
  char *Wa_f, *Wb_f, *Wqkv_f, *Wo_f, *Wgu_f, *Wdown_f;
};

// One layer of a latent-attention model.  Every size is padded with zero weights so that the tile kernels' granularity
// holds for any configuration: Qp, Rp, Fp, EFp are multiples of 64 and a head takes Dp features of q, k, v and gate
// whatever its query/key and value sizes are.
struct LatentLayer {
  rai_hip_latent_layer c;      // the configuration's sizes
  int Qp, Rp, Dp, QD, Fp, EFp; // padded: query rank, latent rank, head, all heads, MLP, expert MLP
  int ldn;                     // Qp + Rp + QD: columns of the down projection's output (query latent | latent | gate)
  char *n1_w, *n2_w, *q_w, *c_w;   // the layer's two norms and the norms of the two latents
  char *Wd;                    // [ldn, Hp]   rows dq | dkv | g, all reading the first norm's output
  char *Wuq;                   // [QD, Qp]
  char *Wkv;                   // [2 QD, Rp]  rows uk | uv
  char *WukT;                  // [heads][Rp][Dp]: uk of each head transposed (built on first use)
  char *Wgu;                   // dense: [2 Fp, Hp] gate / up rows interleaved
  char *Wb;                    // [Hp, QD + Fp]: o | down as one contraction (Fp = 0 without a dense MLP)
  char *Wr;                    // mixture: router [experts, Hp]
  char *We_gu, *We_dn;         // [experts][2 EFp, Hp] interleaved, [experts][Hp, EFp]
  // Wd, Wuq, Wgu, Wb and Wr in MFMA-fragment order for 9 .. 64 rows (built on first use)
  char *Wd_f, *Wuq_f, *Wgu_f, *Wb_f, *Wr_f;
  char *cache;                 // [max_batch][max_context][Rp] normalised latents
};

// Everything a latent-attention decoder has beyond the common fields.
struct LatentModel {
  rai_hip_latent_config c;
  int Hp;                      // width padded to a multiple of 64
  std::vector<LatentLayer> layers;
  float *xs;                   // [max_rows, Hp] residual stream, f32
  char *h1, *h2;               // [max_rows, Hp] outputs of the two norms
  char *dn, *cq, *cn, *q, *kv, *cat;
  char *gathered, *eact, *eout;   // mixture: scaled inputs, activations and outputs, rows sorted by expert
  float *rlogits, *rweight;
  int *rchoice, *rpos;
  MoePlan plan;
  float *ws;                   // partial results of the absorbed attention's context splits
  bool derived_ready;          // WukT matches the loaded parameters
};

// One layer of a hybrid model, padded with zero weights like a latent layer.
struct HybridLayer {
  rai_hip_hybrid_layer c;      // the configuration's sizes
  int Dp, Fp;                  // attention: head width of q, k, v and gate; MLP
  int ldn;                     // columns of the input projection's output
  int QD;                      // columns of the mixer's output: heads * Dp, or heads * Vp
  int a_rank, g_rank;          // padded ranks
  DeltaShape delta;
  char *n1_w;
  char *Wd;                    // [ldn, Hp]  attention: q | k | v | g;  delta rule: q | k | v | b | a1 | g1
  char *Wgu;                   // [2 Fp, Hp] gate / up rows interleaved
  char *Wb;                    // [Hp, QD + Fp]: o | down as one contraction
  char *sink;                  // [heads]
  char *conv, *A_log, *dt_bias, *norm_w, *a2, *g2;   // [channels, taps], [heads], [heads Dk], [Vp], [heads Dk, a_rank], [heads Vp, g_rank]
  const float *cos_t, *sin_t;  // [max_context, rot_dims]
  char *Wd_f, *Wgu_f, *Wb_f, *a2_f, *g2_f;   // in MFMA-fragment order for 9 .. 64 rows (built on first use)
};
// One layer run: a looped layer has one per pass, with what that pass carries from step to step.
struct HybridRun {
  int layer, pass;             // pass >= 0: the first layer of pass `pass`
  char *kcache, *vcache;       // attention: [max_batch][kv_heads][max_context][Dp]
  char *ring;                  // delta rule: the convolutions' last inputs and the state
  float *carried;
};
struct HybridModel {
  rai_hip_hybrid_config c;
  int Hp;
  std::vector<HybridLayer> layers;
  std::vector<HybridRun> runs;
  std::vector<std::pair<RotaryParams, std::pair<const float *, const float *>>> tables;
  char *Wx, *W0, *step;        // loop.in's two halves [Hp, Hp] and [times, Hp]
  char *Wx_f, *W0_f;
  float *xs, *xs2, *x0w;       // [max_rows, Hp]: residual stream (two, swapped by the single-row step's loop entry), W0 x0
  float *stream;               // the one the last forward finished in
  char *h1, *dn, *cat;
  float *decay, *qn, *kn, *beta, *o;   // delta rule, see DeltaArgs
  char *dq, *dk, *dv, *gate, *chunk_ws;
  char *attn_ws;
  int *attn_counters;
  bool derived_ready;          // a padded copy of the embedding table serves as the head
};

}  // namespace rai

using namespace rai;

struct rai_hip_decoder {
  int dev;
  rai_hip_decoder_config cfg;
  size_t es;
  int H, I, QD, KD, D, Hq, Hkv, V, L, NA, KB;
  std::vector<ParamSlot> slots;
  std::map<std::string, int> slot_by_name;
  std::vector<Layer> layers;
  char *embed, *lnf_w, *lnf_b, *head_w, *head_b;
  char *cos_t, *sin_t;  // [max_pos, rot] in the model dtype
  char *kcache, *vcache;
  // activations (sized for max_batch * max_context rows)
  char *x, *x2, *ln, *qkv, *cat, *last, *logits;
  char *attn, *glu;   // sequential block: attention output [rows, QD], gated MLP activation [rows, I]
  char *attn_ws;      // partial results of the decode attention's context splits
  int *attn_counters; // per (batch, head) arrival counters of those splits (zero between launches)
  float embed_scale;  // Gemma: sqrt(hidden) rounded to the model dtype; 1 otherwise
  uint32_t *ids, *tokens, *history;
  char *splitk_ws;        // f32 scratch for prefill GEMMs that split K
  size_t splitk_ws_bytes;
  DevState *state;
  std::vector<void *> allocs;
  int ctx_len;
  int64_t max_rows;
  int history_cap;
  // persistent per-token kernel (Phi-2, bf16, batch 1): per-layer pointer table, exchange packets
  MegaLayer *mega_layers;
  uint64_t *mega_xchg;    // packets exchanged between the blocks of the persistent decode kernel
  unsigned long long *mega_prof;  // time stamps of the persistent kernel when RAI_HIP_MEGA_PROF is set
  bool mega_ok;
  int num_cu;
  hipGraphExec_t step_graph;   // one captured single-token step (batch step_graph_batch)
  hipGraphExec_t step_graph_n; // kGraphSteps consecutive single-token steps in one graph (same batch)
  int step_graph_batch;
  bool x_holds_next;          // d->x already holds the embedding of d->tokens
  // token choice of the example loop (repeat penalty, last maximum wins) instead of plain greedy argmax
  bool sample_on;
  float sample_penalty;
  int sample_last_n;
  uint32_t *token_log;        // [max_batch][token_log_cap]: every token of each sequence so far, prompt first
  int token_log_cap;
  float *choice_val;          // [max_batch][kChoiceMaxSplits]: best value of each share of a wide logits row
  uint32_t *choice_idx;       // and its index
  unsigned long long *head_best;   // one (value, row) word per block of the head kernel that also chooses the token
  char *hidden_copy;          // [max_rows, H]: the residual stream after the last layer, kept when a caller asks for it
  bool want_hidden;           // the running forward copies its final residual stream to hidden_copy
  char *head_f;               // fragment-order copy of the lm_head matrix
  bool frag_ready;            // the fragment-order copies match the loaded parameters
  bool graph_sampled;         // what the cached step graphs were captured with
  float graph_penalty;
  int graph_last_n;
  LatentModel *latent;        // the latent-attention family's part; null for the others
  HybridModel *hybrid;        // the hybrid family's part; null for the others
};


namespace rai {

// decoder.hip: construction and forward pieces every family uses
int dalloc(rai_hip_decoder *d, size_t bytes, char **out);
void add_slot(rai_hip_decoder *d, const std::string &name, int64_t rows, int64_t cols, char *dst, int64_t pitch);
int decoder_embed(rai_hip_decoder *d, hipStream_t st, int64_t rows);
int decoder_linear(rai_hip_decoder *d, hipStream_t st, const LinearArgs &a);
int launch_token_choice(rai_hip_decoder *d, hipStream_t st, int B, int S, bool advance_step);
bool wants_fragments(const rai_hip_decoder *d, int64_t M);
int decoder_fragments(rai_hip_decoder *d, hipStream_t st, char *W, int64_t ldw, int N, int K, char **dst);
void decoder_init_fields(rai_hip_decoder *d, int dev, const rai_hip_decoder_config &cfg);
int decoder_alloc_common(rai_hip_decoder *d);

// decoder_latent.hip
int forward_latent(rai_hip_decoder *d, int B, int S, bool advance_step, bool from_tokens);
// Logits (model dtype, [n, vocab]) of n rows of the residual stream the last forward left; rows_dev: row indices.
int latent_head_rows(rai_hip_decoder *d, hipStream_t st, const int *rows_dev, int n, char *logits);
int latent_hidden_to_host(rai_hip_decoder *d, int64_t rows, float *out);

// decoder_hybrid.hip: the same for the hybrid family
int forward_hybrid(rai_hip_decoder *d, int B, int S, bool advance_step, bool from_tokens);
int hybrid_head_rows(rai_hip_decoder *d, hipStream_t st, const int *rows_dev, int n, char *logits);
int hybrid_hidden_to_host(rai_hip_decoder *d, int64_t rows, float *out);
// device memory that starts as zeros, and a parameter whose rows (columns) come in padded groups (decoder_latent.hip)
int zalloc(rai_hip_decoder *d, size_t bytes, char **out);
void add_grouped_slot(rai_hip_decoder *d, const std::string &name, int64_t rows, int64_t cols, char *dst, int64_t pitch, int64_t row_group,
                      int64_t row_stride, int64_t col_group, int64_t col_stride);
inline int pad64(int n) { return (n + 63) / 64 * 64; }
inline int pad_head(int n) { return n <= 32 ? 32 : n <= 64 ? 64 : n <= 128 ? 128 : n <= 192 ? 192 : n <= 256 ? 256 : pad64(n); }

}  // namespace rai
