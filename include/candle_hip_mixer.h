/*
 * candle_hip_mixer.h — C ABI of the kernels for decoders with unquantized (bfloat16) weights and mixers other than plain
 * causal attention: dense matrix products, windowed attention with kept first tokens and scores mixed across heads,
 * linear attention with a fixed decay per head, and the generalized delta rule.
 *
 * Library libcandle_hip_mixer.so, which also carries the glue of candle_hip_nn.h.  Conventions as in candle_hip_quant.h:
 * device pointers, caller-owned buffers, nothing allocated or synchronized, everything enqueued on `stream`, status codes
 * from enum cq_status.  Activations, caches and recurrent states are f32; weights of matrix products are bfloat16.
 *
 * `pos` is a host integer, `pos_dev` an optional device int32 that is ADDED to it when not NULL: row r of a call has the
 * absolute position pos + *pos_dev + r.  The single-token entry points take both, so a decode step can be captured in a
 * HIP graph.
 */
#ifndef CANDLE_HIP_MIXER_H
#define CANDLE_HIP_MIXER_H

#include <stdint.h>

#include "candle_hip_quant.h"

#ifdef __cplusplus
extern "C" {
#endif

/* ---- dense products -------------------------------------------------------------------------------------------------
 * Weights [n, k] bfloat16, row-major with `ldw` elements per row; k and ldw are multiples of 64 (rows padded with zeros), and
 * activation rows are readable up to k (zero there as well).  CQ_DENSE_BF16 rounds the activations to bfloat16 and
 * accumulates in f32; CQ_DENSE_F32 multiplies in f32 throughout. */
enum cq_dense_precision { CQ_DENSE_BF16 = 0, CQ_DENSE_F32 = 1 };

/* dst[m, n] = x w^T, or dst += x w^T (+ add) with accumulate (the residual stream; `add` is an optional [m, n] addend).
 * ldx, ldd, ld_add: row strides in floats; x 16-byte aligned, ldx % 4 == 0.
 * Few output tiles and a long k are split along k into planes: the workspace holds them (0 bytes when not split). */
int64_t cq_dense_matmul_workspace_bytes(int precision, int64_t m, int64_t n, int64_t k);
int cq_dense_matmul(int precision, const void *w_dev, int64_t ldw, const float *x_dev, int64_t ldx, float *dst_dev, int64_t ldd, const float *add_dev,
                    int64_t ld_add, int accumulate, int64_t m, int64_t n, int64_t k, void *workspace_dev, int64_t workspace_bytes, void *stream);

/* The same product with everything optional that a caller may fold into it.  Zero-initialize, then set what is used (batch = 1 at least).
 *   x_bf16 / dst_bf16   activations / results are bfloat16 (CQ_DENSE_BF16 only; results without accumulate)
 *   act                 applied to the results (without accumulate).  SWIGLU: rows of w alternate gate, up, and silu(gate) * up, n / 2 columns, is stored
 *   row_scale_dev       [m] factors on the stored rows
 *   batch               products side by side: w, x, dst advance by w_batch, x_batch, dst_batch elements (no accumulate, no row factors)
 *   tiles_dev           grouped product: rows [first, first + rows) of tile t meet the weights at w + group * w_batch.  n_tiles_dev [1] tiles exist (at
 *                       most max_tiles; a tile holds at most tile_rows = 32, 64 or 128 rows, 64 for CQ_DENSE_F32); m is the total of rows
 *   src_rows_dev        row r of x is row src_rows[r] in memory;  dst_rows_dev: row r of the result goes to row dst_rows[r] */
typedef struct cq_dense_tile {
    int32_t group, first, rows, reserved;
} cq_dense_tile;
enum cq_dense_act { CQ_DENSE_ACT_NONE = 0, CQ_DENSE_ACT_RELU2 = 1, CQ_DENSE_ACT_SWIGLU = 2 };
typedef struct cq_dense_args {
    const void *w_dev, *x_dev;
    void *dst_dev;
    const float *add_dev, *row_scale_dev;
    const int32_t *src_rows_dev, *dst_rows_dev, *n_tiles_dev;
    const cq_dense_tile *tiles_dev;
    int64_t ldw, ldx, ldd, ld_add, m, n, k, batch, w_batch, x_batch, dst_batch, max_tiles, tile_rows;
    int32_t x_bf16, dst_bf16, accumulate, act;
} cq_dense_args;
int cq_dense_product(int precision, const cq_dense_args *args, void *workspace_dev, int64_t workspace_bytes, void *stream);

/* One activation row, in f32: dst[n] = f(x) w^T (dst += ... (+ add) with accumulate) with f chosen by `prologue`:
 *   CQ_DENSE_PLAIN   f(x) = x
 *   CQ_DENSE_NORM    f(x) = x / sqrt(mean(x^2) + eps) * vec                     (vec [dim])
 *   CQ_DENSE_POLY    f(x) = vec[0] N(x) + vec[1] N(x^2) + vec[2] N(x^3) + vec[3], N(z) = z / sqrt(mean(z^2) + eps)
 *   CQ_DENSE_LAYER_NORM  f(x) = (x - mean(x)) / sqrt(var(x) + eps) * vec[0..dim) + vec[dim..2 dim)
 *   CQ_DENSE_RELU2   f(x) = max(x, 0)^2
 * dim <= k values of x count, f is zero beyond (x is readable up to k, 16-byte aligned).  k <= CQ_DENSE_MATVEC_MAX_K. */
enum cq_dense_prologue { CQ_DENSE_PLAIN = 0, CQ_DENSE_NORM = 1, CQ_DENSE_POLY = 2, CQ_DENSE_LAYER_NORM = 3, CQ_DENSE_RELU2 = 4 };
#define CQ_DENSE_MATVEC_MAX_K 32768
int cq_dense_matvec(const void *w_dev, int64_t ldw, const float *x_dev, int prologue, const float *vec_dev, float eps, int64_t dim, float *dst_dev,
                    const float *add_dev, int accumulate, int64_t n, int64_t k, void *stream);

/* ---- row operations ------------------------------------------------------------------------------------------------
 * RMS norm of selected rows: out[r] = s / sqrt(mean(s^2) + eps) * weight with s = x[index ? index[r] : r] (+ delta[r]); with
 * delta, s also replaces the row of x.  Any dim; strides in floats. */
int cq_mix_rms_norm_rows(float *x_dev, int64_t x_stride, const int32_t *index_dev, const float *delta_dev, int64_t delta_stride, const float *weight_dev,
                         float *out_dev, int64_t out_stride, int64_t rows, int64_t dim, float eps, void *stream);
/* Layer norm of (selected) rows: out[r] = (s - mean(s)) / sqrt(var(s) + eps) * vec[0..dim) + vec[dim..2 dim), s = x[index ? index[r] : r], as f32,
 * as bfloat16 or both (out_dev, out_bf16_dev: one may be NULL). */
int cq_mix_layer_norm_rows(const float *x_dev, int64_t x_stride, const int32_t *index_dev, const float *vec_dev, float *out_dev, void *out_bf16_dev,
                           int64_t out_stride, int64_t rows, int64_t dim, float eps, void *stream);
/* out = coef[0] N(z) + coef[1] N(z^2) + coef[2] N(z^3) + coef[3], N(z) = z / sqrt(mean(z^2) + eps), row by row (out may be z). */
int cq_mix_poly_norm(const float *z_dev, int64_t z_stride, const float *coef_dev, float *out_dev, int64_t out_stride, int64_t rows, int64_t dim, float eps,
                     void *stream);
int cq_mix_tanh(const float *x_dev, int64_t x_stride, float *out_dev, int64_t out_stride, int64_t rows, int64_t dim, void *stream);

/* A group of heads inside a projection row, for the calls below.  Element d of head h of row r is read at
 * src[r * src_stride + src_off + h * dim + d]; an optional RMS norm per head (norm_dev [dim], eps of the call), an optional
 * rotation of the first rot_dims dimensions (pairs (i, i + rot_dims/2); cos/sin [positions, rot_dims/2]) and a factor are applied, and the result goes to
 * dst[h * dst_head_stride + row * dst_row_stride + d], zero for dim <= d < dim_pad.  by_position: `row` is the absolute position
 * (a cache) instead of r.  ctx: rows of the rotation tables and of a cache; positions beyond it are not processed. */
typedef struct cq_mix_heads {
    const float *norm_dev, *cos_dev, *sin_dev;
    float *dst_dev;
    int64_t src_off, dst_row_stride, dst_head_stride;
    int32_t heads, dim, dim_pad, rot_dims, by_position, ctx;
    float factor;
    int32_t reserved;
} cq_mix_heads;
#define CQ_MIX_MAX_GROUPS 6
#define CQ_MIX_MAX_DIM 256
int cq_mix_pack_heads(const float *src_dev, int64_t src_stride, const cq_mix_heads *groups, int n_groups, float eps, const int32_t *pos_dev, int64_t pos,
                      int64_t rows, void *stream);

/* out[r, h * dim + e] = scale * gate(g[r, h * dim + e]) * weight[h * dim + e] * o / sqrt(mean over the head of o^2 + eps).
 * weight optional; gate: CQ_GATE_SILU or CQ_GATE_SIGMOID.  o [rows, heads * dim] with row stride o_stride. */
enum cq_gate { CQ_GATE_SILU = 0, CQ_GATE_SIGMOID = 1 };
int cq_mix_head_norm_gate(const float *o_dev, int64_t o_stride, const float *g_dev, int64_t g_stride, const float *weight_dev, int gate, float scale,
                          float *out_dev, int64_t out_stride, int64_t rows, int64_t heads, int64_t dim, float eps, void *stream);

/* ---- attention with scores mixed across heads, a sliding window and kept first tokens --------------------------------
 * score_h = sum_g talk[h, g] * scale * (q_g . k_g), key j visible to position i when j <= i and (i - j < window or j < keep_first), softmax
 * over the visible keys, out[r, h * vdim + e] = out_scale * sum_j p_h(j) v(j).  Query head h uses kv head h / (n_head / n_kv_head).
 * q [rows, n_head, dim_pad], caches [n_kv_head, ctx, dim_pad] and [n_kv_head, ctx, vdim_pad]; dim_pad and vdim_pad are multiples of 16
 * (padding zero; vdim_pad the least one), at most CQ_MIX_MAX_DIM; n_head <= CQ_MIX_MAX_HEADS.  Calls with few rows split the keys over workgroups and merge
 * through the workspace (0 bytes when not split). */
#define CQ_MIX_MAX_HEADS 64
int64_t cq_mix_talk_attention_workspace_bytes(int64_t rows, int64_t n_head, int64_t vdim, int64_t window, int64_t keep_first, int64_t pos);
int cq_mix_talk_attention(const float *q_dev, const float *k_cache_dev, const float *v_cache_dev, const float *talk_dev, float scale, int64_t window,
                          int64_t keep_first, float out_scale, float *out_dev, int64_t out_stride, int64_t pos, int64_t rows, int64_t n_head,
                          int64_t n_kv_head, int64_t dim_pad, int64_t vdim, int64_t vdim_pad, int64_t ctx, void *workspace_dev, int64_t workspace_bytes,
                          void *stream);

/* The same for one new token straight from its projection row: the three groups (q; k and v with their caches as dst, by_position
 * set) are normalized, rotated and appended as cq_mix_pack_heads would, then attended, in one launch that leaves a record per split of
 * the visible keys in the workspace; the second call merges the records (and runs a retention step beside it, see below). */
int64_t cq_mix_talk_decode_workspace_bytes(int64_t n_head, int64_t vdim, int64_t window, int64_t keep_first, int64_t ctx);
int cq_mix_talk_decode(const float *row_dev, const cq_mix_heads *qkv, float eps, const float *talk_dev, float scale, int64_t window, int64_t keep_first,
                       const int32_t *pos_dev, int64_t pos, void *workspace_dev, int64_t workspace_bytes, void *stream);

/* ---- linear attention with a fixed decay per head (retention) --------------------------------------------------------
 * S <- decay_h S + k v^T, o = S^T q.  States [heads, vdim, state_pad] f32 (column-major S: element (i, j) at [j][i]),
 * state_pad = cq_mix_state_pad(dim), zero at the start of a sequence.  log2_decay_dev [heads]: log2 of the decays.
 * q, k [rows, heads, dim_pad] as cq_mix_pack_heads leaves them; v row r at v_dev + r * v_stride; out raw o [rows, heads * vdim].
 * The rows run as chunks; long calls split into segments that run side by side, joined through the workspace. */
int64_t cq_mix_state_pad(int64_t dim);
int64_t cq_mix_retention_workspace_bytes(int64_t rows, int64_t heads, int64_t dim, int64_t vdim);
int cq_mix_retention(const float *q_dev, const float *k_dev, const float *v_dev, int64_t v_stride, const float *log2_decay_dev, float *state_dev,
                     float *out_dev, int64_t out_stride, int64_t rows, int64_t heads, int64_t dim, int64_t dim_pad, int64_t vdim, void *workspace_dev,
                     int64_t workspace_bytes, void *stream);

/* Second launch of a decode step with the two mixers side by side: merges the records of cq_mix_talk_decode into
 * att_out[n_head * vdim] (times att_scale) and advances the retention states by one token from the same projection row: qk[0], qk[1]
 * describe q and k (dst ignored), v and the gate lie at v_off / g_off; ret_out = ret_scale * silu(g) * o / rms(o). */
int cq_mix_talk_merge_retention_step(const void *workspace_dev, int64_t n_head, int64_t att_vdim, int64_t window, int64_t keep_first, int64_t ctx,
                                     float att_scale, float *att_out_dev, const float *row_dev, const cq_mix_heads *qk, int64_t v_off, int64_t g_off,
                                     const float *decay_dev, float *state_dev, int64_t heads, int64_t vdim, float eps, float ret_scale,
                                     float *ret_out_dev, const int32_t *pos_dev, int64_t pos, void *stream);

/* ---- generalized delta rule -----------------------------------------------------------------------------------------
 * S <- (diag(w) - (a u) u^T) S + k v^T, o = S^T r, u = k / sqrt(sum(k^2) + 1e-6),
 * w = exp(-exp(-1/2) sigmoid(wl + w0)), a = sigmoid(al + a_bias).  States [heads, dim, state_pad], column-major as above.
 * row_dev: projection rows with r, k, v, al at the given offsets (each heads * dim); wl [rows, heads * dim].
 * cq_mix_delta_prep packs w | a u | u | r per (row, head), state_pad floats each, and behind them the |k| = sqrt(sum(k^2) + 1e-6) of every
 * (row, head), rows * heads * (4 state_pad + 1) floats in all, for cq_mix_delta_scan, whose out is the raw o. */
int cq_mix_delta_prep(const float *row_dev, int64_t row_stride, int64_t r_off, int64_t k_off, int64_t a_off, const float *wl_dev, int64_t wl_stride,
                      const float *w0_dev, const float *a_bias_dev, float *packed_dev, int64_t rows, int64_t heads, int64_t dim, void *stream);
int cq_mix_delta_scan(const float *packed_dev, const float *v_dev, int64_t v_stride, float *state_dev, float *out_dev, int64_t out_stride, int64_t rows,
                      int64_t heads, int64_t dim, void *stream);
/* One token, one launch: the low-rank projection of the decay (w2 [heads * dim, rank] bfloat16 with row stride ldw2, applied to tanh of the
 * rank values at low_off), the recurrence, and out = weight * sigmoid(g) * o / rms(o). */
int cq_mix_delta_step(const float *row_dev, int64_t r_off, int64_t k_off, int64_t v_off, int64_t g_off, int64_t a_off, int64_t low_off, const void *w2_dev,
                      int64_t ldw2, int64_t rank, const float *w0_dev, const float *a_bias_dev, const float *weight_dev, float *state_dev, float *out_dev,
                      int64_t heads, int64_t dim, float eps, void *stream);

/* ---- attention over cached latents --------------------------------------------------------------------------------------
 * A position leaves one cache row for all heads: its latent c = rms_norm(z[0..rank), norm) and a rotated key part of rot_dim
 * values (z: its projection row at kv_off).  Per head: key W_uk c beside the rotated part, value W_uv c, causal softmax of
 * (q . k) * scale, the head's output times sigmoid(gate).  Rotation turns dimensions 2i and 2i + 1 together; cos / sin
 * [ctx, rot_dim / 2].
 * Cache rows: rank_pad latent columns (a multiple of 64, zero beyond rank), then rot_pad (a multiple of 8, zero beyond rot_dim) of type T: bfloat16 with
 * `bf16`, else f32.  [ctx] rows; zero-initialize them once.  A projection row holds the queries, head by head [dim unrotated, rot_dim rotated], at 0. */
typedef struct cq_latent {
    const float *norm_dev, *cos_dev, *sin_dev;
    int32_t heads, dim, rot_dim, vdim, rank, rank_pad, rot_pad, ctx, bf16;
    float scale, eps;
    int32_t reserved;
} cq_latent;
#define CQ_LATENT_MAX_RANK 512       /* rank_pad; 256 with rot_pad > 64, which is at most 192 */
#define CQ_LATENT_MAX_HEAD 320       /* dim_pad + rot_pad of the expanded form */
#define CQ_LATENT_MAX_VALUE 256
/* Projection rows into packed queries and, with kv_off >= 0, the cache rows of positions pos ...  Query (r, h) is q[(r * heads + h) * q_head ..] of type T:
 * the rotated part at rot_off, zero up to q_head; the unrotated part in front of it (zero up to rot_off) or, with plain_dev, as f32 at
 * plain[(r * heads + h) * plain_head ..] instead.  Queries come out multiplied by scale * log2(e), which is how the calls below take them. */
int cq_mix_latent_pack(const cq_latent *g, const float *row_dev, int64_t row_stride, int64_t kv_off, void *cache_dev, float *plain_dev, int64_t plain_head, void *q_dev,
                       int64_t q_head, int64_t rot_off, int64_t pos, int64_t rows, void *stream);
/* Attention of rows pos .. pos + rows over keys and values of all heads: kv [pos + rows][kv_row] of type T, head h's unrotated key at h * dim_pad, its value
 * at v_off + h * v_pad (padding of keys zero).  q as packed with rot_off = dim_pad, q_head = dim_pad + rot_pad.  gate row r at gate + r * gate_row, [heads] raw.
 * out[r, h * vdim + e] of type T. */
int cq_mix_latent_expanded(const cq_latent *g, const void *q_dev, int64_t dim_pad, const void *kv_dev, int64_t kv_row, int64_t v_off, int64_t v_pad, const void *cache_dev,
                           const float *gate_dev, int64_t gate_row, void *out_dev, int64_t out_row, int64_t pos, int64_t rows, void *stream);
/* The same over the cache rows themselves: q [rows][heads][rank_pad + rot_pad] holds W_uk^T q beside the rotated part; out [rows][heads][rank_pad] f32 is the
 * attended latent times the gate, which W_uv takes to the head's output.  Few queries split the keys and merge through the workspace (0 bytes
 * when not split).  step: the workspace of cq_mix_latent_step. */
int64_t cq_mix_latent_absorbed_workspace_bytes(const cq_latent *g, int64_t rows, int64_t pos, int step);
int cq_mix_latent_absorbed(const cq_latent *g, const void *q_dev, const void *cache_dev, const float *gate_dev, int64_t gate_row, float *out_dev, int64_t pos, int64_t rows,
                           void *workspace_dev, int64_t workspace_bytes, void *stream);
/* One new token from its projection row to the gated head outputs [heads * vdim], three launches: w_ukt [heads][rank][ld_ukt] (W_uk transposed head by head) and
 * w_uv [heads * vdim][ld_uv] bfloat16, zero beyond dim and rank; gate at row + gate_off; q_dev: scratch of heads * (rank_pad + rot_pad) T, zero-initialized once. */
int cq_mix_latent_step(const cq_latent *g, const float *row_dev, int64_t kv_off, void *cache_dev, const void *w_ukt_dev, int64_t ld_ukt, const void *w_uv_dev, int64_t ld_uv,
                       int64_t gate_off, void *q_dev, float *out_dev, const int32_t *pos_dev, int64_t pos, void *workspace_dev, int64_t workspace_bytes, void *stream);

/* ---- mixture of experts ------------------------------------------------------------------------------------------------
 * cq_mix_moe_select  ids / weights [rows, top]: the `top` largest of the `experts` router logits of a row, largest first (equals: lower id first), and the softmax
 *                    over those chosen.  shared_weights (optional) [rows]: sigmoid of the logit behind the experts'.
 * cq_mix_moe_plan    the pairs (row, choice) gathered by expert for a grouped product: gathered row i is row src_rows[i] of the input and pair
 *                    dst_rows[i] = row * top + choice, its weight scale[i]; tiles of at most tile_rows of them, n_tiles[0] of cq_mix_moe_max_tiles.
 *                    The order of an expert's pairs is unspecified.
 * cq_mix_moe_add     x[r] += y[r * top] + ... + y[r * top + top - 1] */
#define CQ_MOE_MAX_EXPERTS 1024
#define CQ_MOE_MAX_TOP 64
int cq_mix_moe_select(const float *logits_dev, int64_t ld, int64_t rows, int64_t experts, int64_t top, int32_t *ids_dev, float *weights_dev, float *shared_weights_dev,
                      void *stream);
int64_t cq_mix_moe_max_tiles(int64_t rows, int64_t experts, int64_t top, int64_t tile_rows);
int cq_mix_moe_plan(const int32_t *ids_dev, const float *weights_dev, int64_t rows, int64_t experts, int64_t top, int64_t tile_rows, int32_t *src_rows_dev,
                    int32_t *dst_rows_dev, float *scale_dev, cq_dense_tile *tiles_dev, int32_t *n_tiles_dev, void *stream);
int cq_mix_moe_add(const float *y_dev, int64_t ldy, int64_t top, float *x_dev, int64_t ldx, int64_t rows, int64_t dim, void *stream);
/* One token: x += sum of weight_e W_down,e (silu(W_gate,e f(x)) * (W_up,e f(x))) over the chosen experts, plus sigmoid(logits[experts]) times the shared one
 * (shared_ff > 0), plus `add`, with f the norm CQ_DENSE_NORM or CQ_DENSE_LAYER_NORM (vec, eps).  Two launches; the choice is part of the first.
 * Weights bfloat16: up [2 ff][kp] per expert, rows alternating gate and up; down [dim][ffp]; zero beyond dim and ff.  act_dev: top * ffp + shared_ffp
 * floats, ids_dev: top ints of scratch.  cq_mix_moe_step_fits: whether the sizes fit the launches (else CQ_ERR_RANGE). */
typedef struct cq_moe {
    const void *up_dev, *down_dev, *shared_up_dev, *shared_down_dev;
    int64_t up_stride, down_stride;          /* weights from one expert to the next */
    int32_t experts, top, kp, ff, ffp, shared_ff, shared_ffp, reserved;
} cq_moe;
int cq_mix_moe_step_fits(const cq_moe *g);
int cq_mix_moe_step(const cq_moe *g, float *x_dev, int norm, const float *vec_dev, float eps, int64_t dim, const float *logits_dev, float *act_dev, int32_t *ids_dev,
                    const float *add_dev, void *stream);

#ifdef __cplusplus
}
#endif
#endif
