/*
 * ughip_layers.h -- the layer mechanisms of decoders beyond llama, as entry points of libughip.so: products of rows of any
 * size with their neighbours folded in, RMS norms on a sublayer's output, latent attention, a state-space recurrence with
 * its causal convolution, routed experts, and per-layer token inputs.  None of them has a counterpart in ug-llama
 * (ug-llama/src/main.rs:22-28); the conventions (error codes, element counts, one stream) are those of ughip.h.
 *
 * Activations are F32.  Matrices are row-major [out, in], F32 or BF16.  A `ughip_view` is m rows inside a slice: row i
 * starts at element offset + i * stride.  Every size is an argument and every access is checked against the slices on the
 * host before a launch.
 */
#ifndef UGHIP_LAYERS_H_
#define UGHIP_LAYERS_H_

#include "ughip.h"

#ifdef __cplusplus
extern "C" {
#endif

typedef struct ughip_view {
  ughip_slice* s; /* NULL: absent */
  size_t offset, stride;
} ughip_view;

/* (Results called F32 or BF16 below take the dtype of their slice.)
 * dst[i, :] = table[ids[i], col .. col + cols), table F32 or BF16 with rows of `stride` elements (an embedding lookup, or the
 * part of one that belongs to a layer).  Ids outside [0, table_rows) give NaN rows and read nothing.
 * dst F32 or BF16. */
int ughip_gather_rows(ughip_device* dev, const ughip_slice* table, size_t table_rows, size_t stride, size_t col, size_t cols,
                      const ughip_slice* ids, size_t m, ughip_view dst);

/* ---- products of rows ---------------------------------------------------------------------------------------------------
 * dst = act(x w^T + bias), any m, n, k.  `product`:
 *   UGHIP_PRODUCT_F32   x and w F32, the f32 matrix pipe;
 *   UGHIP_PRODUCT_BF16  x and w rounded to (or stored as) bf16, the bf16 matrix pipe, f32 accumulation.  (2 .. 128 dense F32 rows
 *                       against a BF16 matrix of regular sizes keep their F32 values: the kernels of ughip_linear_rows.)
 * x, w and dst may each be F32 or BF16 (F32 only for UGHIP_PRODUCT_F32).  BF16 rows and matrices of regular sizes take the
 * one-wave-per-SIMD kernel of ughip_matmul, the rest one that takes any size (ughip_last_kernel names it).
 * `act`:
 *   UGHIP_ACT_NONE      dst[m, n] = y;
 *   UGHIP_ACT_SWIGLU    w is [2 n, k], gate rows then up rows (and bias 2 n values): dst = silu(y_gate) * y_up;
 *   UGHIP_ACT_GLU       as SWIGLU with another gated unit: dst = g * sigmoid(act_alpha g) * (u + act_shift), where with act_limit > 0
 *                       g = min(y_gate, act_limit) and u = y_up kept within +- act_limit;
 *   UGHIP_ACT_GELU_MUL  dst[i, c] = gelu_tanh(y[i, c]) * table[ids[i], table_col + c]: a gate whose other factor is a table row
 *                       chosen by the row's token.
 * groups > 0: w holds `groups` matrices one after the other and the m rows come sorted by group: rows
 * group_end[g - 1] .. group_end[g] - 1 meet matrix g, and row r reads x row row_index[r] (NULL: r); what ughip_group_rows
 * writes.  No bias then. */
enum { UGHIP_PRODUCT_BF16 = 2 };
enum { UGHIP_ACT_NONE = 0, UGHIP_ACT_SWIGLU = 1, UGHIP_ACT_GELU_MUL = 2, UGHIP_ACT_GLU = 3 };
typedef struct ughip_product {
  ughip_view x, dst;
  const ughip_slice *w, *bias;
  size_t w_stride; /* elements from one row of w to the next, 0: k (plain form only) */
  size_t m, n, k;
  int product, act;
  const ughip_slice *table, *ids;
  size_t table_rows, table_stride, table_col;
  const ughip_slice *row_index, *group_end;
  size_t groups, x_rows; /* x_rows: rows of x when row_index is given */
  float act_alpha, act_shift, act_limit; /* UGHIP_ACT_GLU */
} ughip_product;
int ughip_product_rows(ughip_device* dev, const ughip_product* p);

/* ---- norms --------------------------------------------------------------------------------------------------------------
 * dst[i] = x[i] + y[i] / sqrt(mean(y[i]^2) + eps) * w: a sublayer's normed output joins the residual (x.s NULL: the norm
 * alone).  y may be the sum of `top` rows: y[i] = sum_j weights[i top + j] * y.row(slots[i top + j]) (routed experts, summed
 * in the order j).  y.s NULL: nothing is normed, w is not read.  extra (may be absent): rows that join as they are.
 * dst may be x, and may be BF16; copy (may be NULL, F32 or BF16): dense rows [m, n] of the result once more, or with `next` of
 * result / sqrt(mean(result^2) + eps) * next, the norm in front of the next sublayer.  n <= 16000. */
int ughip_add_rms_norm_rows(ughip_device* dev, ughip_view x, ughip_view y, const ughip_slice* slots, const ughip_slice* weights, size_t top, size_t y_rows,
                            const ughip_slice* w, float eps, ughip_view extra, ughip_view dst, const ughip_slice* next, ughip_slice* copy, size_t m, size_t n);
/* dst[i] = g / sqrt(mean(g^2) + eps) * w with g = y[i] * silu(z[i]), the mean taken over each of `groups` equal parts of the
 * row on its own.  z.s NULL: g = y.  dst F32 or BF16. */
int ughip_gated_rms_norm_rows(ughip_device* dev, ughip_view y, ughip_view z, const ughip_slice* w, float eps, size_t groups, ughip_view dst, size_t m, size_t n);

/* ---- latent attention -----------------------------------------------------------------------------------------------------
 * The cache of a layer is [cap, rank + rot] F32 rows: the normed latent, then the rotated key part all heads share.  Rotation
 * is the 'rotate half' pairing over the whole rot part, angles from tables cos, sin [table_rows, rot / 2] at row = position.
 * ughip_latent_append: rows kv [t, rank + rot] of a projection become cache rows pos .. pos + t - 1: the first `rank`
 *   elements / sqrt(mean^2 + eps) * w, the rest rotated. */
int ughip_latent_append(ughip_device* dev, ughip_view kv, const ughip_slice* w, float eps, const ughip_slice* cos, const ughip_slice* sin, size_t table_rows,
                        ughip_slice* cache, size_t cap, size_t pos, size_t t, size_t rank, size_t rot);
/* Causal attention of t positions pos .. pos + t - 1 over cache rows 0 .. pos + t - 1 with keys and values expanded from the
 * latents: q rows [t, heads (dim + rot)] (not yet rotated), k [pos + t, heads dim], v_t [heads vdim, v_stride] (values
 * transposed: one row per value element, position along it), both F32 or both BF16; dst [t, heads vdim] F32 or BF16.  With BF16
 * operands q is rounded to bf16, scores and weights stay f32 (a weight meets v as two bf16 terms). */
int ughip_latent_attention_rows(ughip_device* dev, ughip_view q, const ughip_slice* k, const ughip_slice* v_t, size_t v_stride, const ughip_slice* cache,
                                const ughip_slice* cos, const ughip_slice* sin, size_t table_rows, ughip_view dst, size_t t, size_t pos, size_t heads, size_t dim,
                                size_t rot, size_t vdim, size_t rank, float scale);
/* The same for few positions without expanding anything: the heads' up-projections are folded into the query and the result
 * (w_uk [heads dim, rank], w_uv [heads vdim, rank]), every head attends to the latents themselves.  All in f32.
 * kv given: the step's rows are appended to the cache (cap rows) on the way, as ughip_latent_append does with (kv, kv_norm, eps). */
int ughip_latent_attention_absorbed(ughip_device* dev, ughip_view q, ughip_view kv, const ughip_slice* kv_norm, float eps, const ughip_slice* w_uk,
                                    const ughip_slice* w_uv, ughip_slice* cache, size_t cap, const ughip_slice* cos, const ughip_slice* sin, size_t table_rows,
                                    ughip_view dst, size_t t, size_t pos, size_t heads, size_t dim, size_t rot, size_t vdim, size_t rank, float scale);

/* ---- grouped attention ----------------------------------------------------------------------------------------------------
 * Causal attention of t positions pos .. pos + t - 1 from projected rows qkv [t, heads dim | kv_heads dim | kv_heads vdim] (F32): query
 * head h reads key / value head h / (heads / kv_heads).  The first `rot` elements of queries and keys are rotated in neighbouring pairs
 * (2 i, 2 i + 1), angles from tables cos, sin [table_rows, rot / 2] at row = position (rot 0: none); queries are multiplied by
 * q_factor[position] (NULL: 1).  window > 0: a position sees itself and the window - 1 positions in front of it; 0: all of them.
 * The step's keys and values join the caches, F32 or BF16 (then products run on bf16 operands; scores and weights stay f32): buffers
 * of the sizes ughip_grouped_attention_cache gives for `capacity` positions, the layout is the library's.  dst [t, heads vdim] F32 or
 * BF16.  dim and vdim are at most 256. */
typedef struct ughip_attention {
  ughip_view qkv, dst;
  ughip_slice *k_cache, *v_cache;
  const ughip_slice *cos, *sin, *q_factor;
  size_t capacity, table_rows, rot, window;
  size_t t, pos, heads, kv_heads, dim, vdim;
  float scale;
} ughip_attention;
int ughip_grouped_attention(ughip_device* dev, const ughip_attention* p);
/* rows: what `capacity` is rounded up to. */
int ughip_grouped_attention_cache(size_t kv_heads, size_t dim, size_t vdim, size_t capacity, size_t* rows, size_t* k_elems, size_t* v_elems);

/* ---- a state-space recurrence behind a causal convolution ------------------------------------------------------------------
 * ughip_conv_silu_rows: dst[i, c] = silu(bias[c] + sum_j taps[c, j] x[i - (n_taps - 1) + j, c]) for t positions from `pos` on;
 *   rows before the step come from `ring` [n_taps, channels] (row p at p % n_taps), rows before position 0 are zeros.
 * ughip_conv_ring_store: the step's last rows go into the ring (after everything that still reads the old ones). */
int ughip_conv_silu_rows(ughip_device* dev, ughip_view x, const ughip_slice* taps, const ughip_slice* bias, size_t n_taps, const ughip_slice* ring, size_t pos,
                         size_t t, size_t channels, ughip_view dst);
int ughip_conv_ring_store(ughip_device* dev, ughip_view x, size_t n_taps, ughip_slice* ring, size_t pos, size_t t, size_t channels);
/* xbc rows [heads vdim | groups state (B) | groups state (C)] (after the convolution), dt rows [heads] as projected:
 *   d = softplus(dt + dt_bias), S_h = exp(-exp(a_log_h) d_h) S_h + d_h B_g x_h^T, y_h = S_h^T C_g + skip_h x_h, g = h / (heads / groups)
 * for t positions; s [heads, state, vdim] F32 is read (as zeros when pos == 0) and left at its last value.  dst [t, heads vdim].
 * Several positions run as chunks: the products inside a chunk on the f32 matrix pipe, a scan over the chunks' states. */
int ughip_ssm_rows(ughip_device* dev, ughip_view xbc, ughip_view dt, const ughip_slice* dt_bias, const ughip_slice* a_log, const ughip_slice* skip, ughip_slice* s,
                   size_t pos, size_t t, size_t heads, size_t vdim, size_t groups, size_t state, ughip_view dst);

/* ---- a gated delta rule with a decay per key channel ------------------------------------------------------------------------
 * Per head h, with keys and queries of head h / (heads / kv_heads), a state s_h [dim, vdim] and everything in f32:
 *   k = unit(k), q = unit(q) / sqrt(dim), unit(x) = x / sqrt(sum(x^2) + 1e-6);  beta = sigmoid(b_h)
 *   decay_c = exp(-exp(a_log_h) softplus(a_hc + dt_bias_hc)) for every key channel c
 *   s = decay * s;  u = beta (v - s^T k);  s = s + k u^T;  o = s^T q
 * The state is read (as zeros when pos == 0) and left at its last value.
 * ughip_delta_rows: t positions, rows qkv [t, kv_heads dim (q) | kv_heads dim (k) | heads vdim (v)] behind the convolution
 *   (ughip_conv_silu_rows), b [t, heads], a [t, heads dim], and the output leaves normed and gated:
 *   dst[i] = o / sqrt(mean(o^2) + eps) * norm * sigmoid(z), per head, norm [vdim], z and dst [t, heads vdim] (dst F32 or BF16).
 *   Several positions run as chunks: a triangular solve inside each, a scan over the chunks' states.
 * ughip_delta_step: one position from its projected row p = [.. qkv (at qkv_offset) .. b .. a_in (a_rank) .. z_in (z_rank)], the
 *   convolution with its ring (ughip_conv_silu_rows, ughip_conv_ring_store) included, a = w_a a_in, z = w_z z_in (matrices
 *   [heads dim, a_rank] and [heads vdim, z_rank], F32 or BF16).  dst (at dst_offset): o [heads vdim], then z [heads vdim].
 * dim and vdim are at most 256. */
typedef struct ughip_delta {
  size_t t, pos, heads, kv_heads, dim, vdim;
  const ughip_slice *a_log, *dt_bias, *norm;
  ughip_slice* s;
  float eps;
  ughip_view qkv, b, a, z, dst; /* rows */
  const ughip_slice* p;         /* step */
  size_t qkv_offset, b_offset, a_offset, z_offset, a_rank, z_rank, n_taps, dst_offset;
  const ughip_slice *taps, *w_a, *w_z;
  ughip_slice *ring, *out;
} ughip_delta;
int ughip_delta_rows(ughip_device* dev, const ughip_delta* p);
int ughip_delta_step(ughip_device* dev, const ughip_delta* p);

/* ---- routed experts ------------------------------------------------------------------------------------------------------
 * Scores s = sigmoid(x router^T) in f32; choice scores s + correction; the experts form `groups` runs of equal size, a run's
 * score is the sum of its two largest choice scores, the `keep` best runs stay; the `top` best choice scores among them are
 * chosen (equal scores: the lower index).  ids[i top + j] = expert, weights[i top + j] = s of it. */
int ughip_route_rows(ughip_device* dev, ughip_view x, const ughip_slice* router, const ughip_slice* correction, size_t m, size_t k, size_t experts, size_t groups,
                     size_t keep, size_t top, ughip_slice* ids, ughip_slice* weights);
/* ids [m top] -> the (row, choice) pairs sorted by expert, rows in order within one: row_index[r] = row, slots[i top + j] = r,
 * group_end[e] = number of pairs with an expert <= e. */
int ughip_group_rows(ughip_device* dev, const ughip_slice* ids, size_t m, size_t top, size_t experts, ughip_slice* row_index, ughip_slice* slots,
                     ughip_slice* group_end);

/* ---- one position ---------------------------------------------------------------------------------------------------------
 * A product of one row with what stands in front of it folded into the launch.  The row the matrix meets is made in every
 * workgroup while the matrix is on its way:
 *   v = x                                                     (k values)
 *   v = x + y / sqrt(mean(y^2) + eps) * y_norm (+ extra)      y given: a sublayer's output joins the residual; v also goes to
 *                                                             dst at x_out (keep_x)
 *   v = x * silu(gate)                                        gate given
 *   v = v / sqrt(mean(v^2) + eps) * norm                      norm given, the mean over each of norm_groups equal parts
 *   v = v * sigmoid(gate)                                     gate given with gate_after (instead of silu(gate) above)
 * Then dst[dst_offset ..] = act(v w^T + bias) as in ughip_product_rows (n columns, w F32 or BF16, sums in f32).
 * Routed experts: route != 0, w holds `experts` matrices one after the other.
 *   route == 1: the choice is made from router logits (in every workgroup; the first one leaves ids and weights), and the
 *     result is one run of n columns per chosen expert, top n in all;
 *   route == 2: ids and weights are read, x holds one row of k per chosen expert (top k values), and the result is the weighted
 *     sum of the experts' products: n columns.
 * The input row, every expert's part rounded up to a multiple of 512, has at most 16384 elements. */
typedef struct ughip_row_step {
  const ughip_slice* x;
  size_t x_offset;
  const ughip_slice *y, *y_norm, *gate, *norm;
  size_t y_offset, gate_offset, norm_groups;
  float eps;
  int act, route, keep_x;
  const ughip_slice *w, *bias;
  size_t n, k;
  const ughip_slice *table, *ids; /* UGHIP_ACT_GELU_MUL: ids[0] is the row's token */
  size_t table_rows, table_stride, table_col;
  const ughip_slice *logits, *correction;
  size_t logits_offset, experts, groups, keep, top;
  ughip_slice *route_ids, *route_weights;
  ughip_slice* dst;
  size_t dst_offset, x_out;
  const ughip_slice* extra;
  size_t extra_offset;
  int gate_after;
  float act_alpha, act_shift, act_limit; /* UGHIP_ACT_GLU */
} ughip_row_step;
int ughip_product_row(ughip_device* dev, const ughip_row_step* p);
/* One position of the state-space mixer from the projected row p = [.. | x | B | C (at xbc_offset) | dt (at dt_offset)]:
 * ughip_conv_silu_rows, ughip_conv_ring_store and ughip_ssm_rows for t = 1 in one launch. */
int ughip_ssm_step(ughip_device* dev, const ughip_slice* p, size_t xbc_offset, size_t dt_offset, const ughip_slice* taps, const ughip_slice* conv_bias,
                   size_t n_taps, ughip_slice* ring, const ughip_slice* dt_bias, const ughip_slice* a_log, const ughip_slice* skip, ughip_slice* s, size_t pos,
                   size_t heads, size_t vdim, size_t groups, size_t state, ughip_view dst);

#ifdef __cplusplus
}
#endif
#endif /* UGHIP_LAYERS_H_ */
