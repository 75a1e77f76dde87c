// Launchers of the latent-attention family's kernels: norms of an f32 residual stream (norm.hip), attention
// over cached latents (latent_attention.hip) and the mixture of experts (moe.hip).  `dtype` is RAI_BF16 or RAI_F32
// throughout; "T" below stands for its storage type.
#pragma once
#include "common.h"
#include "decode_mega.h"
#include "gemm.h"

namespace rai {

// Row r of the output is row first + r * step of the stream.  The row is src (f32 stream or T rows) plus
//   add_scale * sum_j add[add_rows[row * top + j], :]
// (the pending outputs of a mixture), times src_scale, is written back to `x` when given, and is normalised in `groups`
// equal runs, each by its own 1 / sqrt(mean square + eps); h1 = normalised * w1 * h_scale and, when given,
// h2 = normalised * w2 * h_scale.  kStreamLayerNorm: one run, and its mean is taken off first.  kStreamCopy: not
// normalised at all, no weights.
enum StreamNormKind { kStreamRms = 0, kStreamLayerNorm = 1, kStreamCopy = 2 };
struct StreamNormArgs {
  const void *src;
  int src_f32;
  int64_t src_ld;
  float *x;            // f32 stream, may be src itself; null: not written back
  int64_t x_ld;
  const void *add;     // T rows; null: none
  const int *add_rows;
  int64_t add_ld;
  int top;
  float add_scale;
  const void *w1, *w2;
  void *h1, *h2;       // dense rows, h_ld apart; columns [width, h_ld) are set to zero
  int64_t h_ld;
  int width, groups;
  float eps;
  int64_t rows, first, step;
  const int *row_map;  // explicit stream row of each output row instead of first + r * step
  int kind;            // StreamNormKind
  float src_scale, h_scale;   // 0 stands for 1
};
int launch_stream_norm(hipStream_t st, int dtype, const StreamNormArgs &a);

// ---- latent attention.  A layer caches one normalised latent c[Rp] per token; head h's key and value are
// uk[h] c and uv[h] c.
// Norm of the two latents of a down-projection row [query latent (Qp) | latent (Rp) | gate]: cq = norm(row[0, q_rank)) and
// the cache row of position pos + s = norm(row[Qp, Qp + kv_rank)), also written to cn when given.  Padding stays zero.
struct LatentNormArgs {
  const void *dn;
  int64_t ldn;
  int q_rank, Qp, kv_rank, Rp;
  const void *q_w, *c_w;
  void *cq, *cn, *cache;     // [rows, Qp], [rows, Rp] or null, [B][Tmax][Rp]
  const DevState *state;
  int B, S, Tmax;
  float eps;
};
int launch_latent_norm(hipStream_t st, int dtype, const LatentNormArgs &a);

// The absorbed form, for few query rows: qa[row, h] = uk[h]^T q[row, h] meets the cached latents directly, the weighted
// sum of latents goes through uv[h] and the output gate.
struct LatentAttnArgs {
  const void *q;             // [rows, heads * Dp]
  const void *WukT;          // [heads][Rp][Dp]
  const void *Wuv;           // [heads * Dp, Rp]
  const void *cache;         // [B][Tmax][Rp]
  const void *gate;          // row stride ldg, head h feature d at h * Dp + d
  int64_t ldg;
  void *out;                 // row stride ldo, same feature order
  int64_t ldo;
  void *qa;                  // scratch [rows, heads, Rp] of T
  float *ws;                 // scratch, latent_attn_ws_floats()
  const DevState *state;     // row (b, s) is position state->pos + s
  int B, S, heads, Dp, Rp, Tmax, window;
  float scale;
  int splits;                // filled in by the launcher
};
size_t latent_attn_ws_floats(int rows, int heads, int Rp);
int launch_latent_attention(hipStream_t st, int dtype, LatentAttnArgs a);
// WukT[h][r][d] = Wuk[h * Dp + d][r]
int launch_latent_transpose_uk(hipStream_t st, int dtype, const void *Wuk, void *WukT, int heads, int Dp, int Rp);

// ---- the single-row bf16 step (latent_decode.hip): launches with norms, routing, append and residual folded in.  The
// hybrid family's step uses the first and the last of them.
struct LatentInArgs {
  const void *src;              // the stream row, f32 or (first layer) the bf16 embedding row
  int src_f32;
  int H, groups, K;             // width, norm groups, padded width
  float eps;
  int64_t ldw;
  int kind;                     // StreamNormKind; kStreamCopy: no norm, n1 and n2 are not read
  float src_scale, h_scale;     // 0 stands for 1: what the source and the norm's output are multiplied with
  const void *W1, *n1;          // rows on the first norm's output -> bf16
  int N1;
  void *out1;
  const void *W2, *n2;          // rows on the second norm's: gated pairs -> bf16 out2[n / 2], or plain -> f32 out2[n]
  int N2, gated2, act;
  float act_limit, act_alpha;   // kActClampedGlu
  const float *add2;            // plain form: out2[n] = product + add2[n] + bias2[n], either may be null
  const void *bias2;
  void *out2;
  void *h2;                     // the second norm's output, for the experts; null: not kept
  int waves1, rows_per_wave;    // filled in by the launcher
};
int launch_latent_in(hipStream_t st, LatentInArgs a);
struct LatentMidArgs {
  const void *dn;               // [query latent (Qp) | latent (Rp) | gate]
  int q_rank, Qp, kv_rank, Rp;
  const void *q_w, *c_w;
  float eps;
  const void *Wuq;              // [Nq, Qp] -> q
  int Nq;
  void *q;
  void *cache;                  // [Tmax, Rp], row state->pos is written
  const DevState *state;
  const float *rlogits;         // mixture (top > 0): router logits, gated rows of the chosen experts -> eact [top, EFp]
  int experts, top;
  const void *h2, *We_gu;
  int Hp, EFp, act;
  int64_t gu_stride;
  void *eact;
  int *choice;
  int waves_q, waves_e, rows_per_wave;   // filled in by the launcher
};
int launch_latent_mid(hipStream_t st, LatentMidArgs a);
// Few rows of a mixture: gated rows of every slot's expert on weight[slot] * h[slot / top] -> eact [slots, EFp]
struct MoeSlotsArgs {
  const void *h;                // [tokens] rows, ld apart
  int64_t ld;
  int slots, top;
  const int *choice;
  const float *weight;
  const void *We_gu;
  int Hp, EFp, act;
  int64_t gu_stride;
  void *eact;
  int waves_e, rows_per_wave;   // filled in by the launcher
};
bool moe_slots_serves(int64_t slots, int experts, int Hp, int top, int EFp);
int launch_moe_slots(hipStream_t st, MoeSlotsArgs a);
// For each of `rows` rows (x0, x1, choice, res and out dense, row by row):
// out[n] = res[n] + mult * (W0[n] . x0 + sum_j W1[choice[j]][n] . x1[j]); rows of W0 (W1) are K0 (K1) long
struct LatentDownArgs {
  const void *x0, *W0;
  int K0;
  const void *x1, *W1;
  int K1, top;
  int64_t stride1;
  const int *choice;
  const void *res;
  int res_f32, H, N, rows;
  float res_scale;   // 0 stands for 1
  float mult;
  float *out;
};
int launch_latent_down(hipStream_t st, const LatentDownArgs &a);
bool latent_single_row_serves(int width, int groups, int max_rank, int max_experts, int64_t down_columns);

// ---- mixture of experts
// Device-side plan of one mixture: the (token, choice) slots sorted by expert, cut into row tiles of `bm`.
struct MoePlan {
  int4 *tiles;     // {expert, first sorted row, rows, 0}
  int *n_tiles;    // device count
  int *slot_of;    // sorted row -> slot
  int *counts;     // scratch, moe_plan_counts()
  int cap_tiles;
};
int moe_max_tiles(int64_t slots, int experts, int bm);
constexpr int64_t kPlanFewSlots = 8192;   // up to here the plan is one launch
constexpr int kPlanExperts = 2048;
int64_t moe_plan_counts(int64_t slots, int experts);   // ints
// choice[t * top + j], weight[t * top + j]: the `top` largest sigmoid scores of the token's logits, in decreasing order.
int launch_moe_route(hipStream_t st, const float *logits, int64_t tokens, int experts, int top, int *choice, float *weight);
int launch_moe_plan(hipStream_t st, const int *choice, int64_t slots, int experts, int bm, const MoePlan &plan, int *row_of_slot);
// out[r] = weight[slot] * h[slot / top], slot = slot_of[r]
int launch_moe_gather(hipStream_t st, int dtype, const void *h, int64_t ld, int cols, const MoePlan &plan, const float *weight, int top,
                      int64_t slots, void *out);
// One Linear per expert over its rows of the sorted order: W of expert e is w_stride elements behind that of e - 1.
constexpr int kGroupedRowsBf16 = 128, kGroupedRowsF32 = 64;   // smallest row tile (`bm` of the plan) of the two forms
int linear_grouped_rows(int dtype, int64_t slots, int experts);   // the row tile to plan for
int launch_linear_bf16_grouped(hipStream_t st, const LinearArgs &a, int64_t w_stride, const MoePlan &plan, int bm);
int launch_linear_f32_grouped(hipStream_t st, const LinearArgs &a, int64_t w_stride, const MoePlan &plan);

}  // namespace rai
