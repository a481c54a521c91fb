/* tah_mixers.h -- C ABI of the layer mechanisms of decoder models that are described layer by layer: residual rows
 * with norms around the sublayers, short convolutions of a sublayer's input, gated delta-rule recurrence, sliding-window
 * attention on latents or on keys and values, mixture of experts.  Same conventions as tah_duo.h (device pointers, nothing
 * allocated, nothing synchronised, 0 or TAH_E_*), exported by the same library.  Sizes and constants are arguments; nothing
 * here belongs to one model.
 *
 * Element type.  `dtype` says what activations, weights and cached rows are: TAH_DT_BF16 or TAH_DT_F32.  The residual
 * rows, norms, attention scores and weights, router logits and recurrent state are float32 with either.
 *
 * Padding.  Row-major activations carry padded columns (the matrix kernels work in steps of 32): a padded column holds
 * zero, and zero columns of the next weight meet it.  `cols` is the padded width of a row, `width` the true one.
 *
 * Sequences.  A portion of sequence b is rows [cu[b], cu[b+1]) of the packed rows; it belongs to state slot slot[b]
 * and starts at position pos0[b].  A portion at position 0 reads nothing of its slot (whatever an earlier owner left
 * there), so a slot is reset by starting over.  A negative slot (or, for single rows, position) drops the row: nothing
 * is read from or written to any slot for it. */
#ifndef TAH_MIXERS_H
#define TAH_MIXERS_H

#include "tah_duo.h"

#ifdef __cplusplus
extern "C" {
#endif

enum { TAH_DT_BF16 = 0, TAH_DT_F32 = 1 };

typedef struct tah_portions {
    const int32_t *cu, *slot, *pos0; /* [nseq + 1], [nseq], [nseq] */
    const int32_t* row_seq;          /* [rows] */
    int32_t nseq, rows;
} tah_portions;

/* ---- residual rows ------------------------------------------------------------------------------------------- */

/* x = scale * embed[tok], in float32, in the element type and (rows <= 32) in the rows form of tah_linear_rows; and the rows'
 * slots and positions for a decode step: row r owns slot slot_base + r, finished rows get -1. */
typedef struct tah_embed_rows_args {
    const int64_t* tok;       /* [rows], clamped into the vocabulary */
    const int32_t* pos;       /* [rows] or NULL (then slot / q_pos / active are not written) */
    const uint8_t* finished;  /* [rows] or NULL */
    const void* embed;        /* [vocab, cols] */
    float* x;                 /* [rows, cols] */
    void* xe;                 /* [rows, cols] in the element type, or NULL */
    void* x_packed;           /* bf16 rows form [32 * cols], or NULL */
    int32_t *slot, *q_pos;    /* [rows] */
    uint8_t* active;          /* [rows] */
    int32_t rows, vocab, cols, dtype, slot_base;
    float scale;
} tah_embed_rows_args;
int tah_embed_rows(const tah_embed_rows_args* args, tah_stream_t stream);

/* x += coef * y / sqrt(mean(y^2) + eps): the norm of a sublayer's output, its weight and any layer scale in `coef`, and
 * the residual sum, all in float32.  y = y_scale[r] * y[r] + sum_j weight[r][j] * experts[index[r][j] * index_scale +
 * r * index_row] (either part may be absent; without both, x stays as it is).  Optionally, from the new x: its row in the
 * element type and in rows form, and a norm of it, n = next_coef * x / sqrt(mean(x^2) + eps), as the next sublayer's (or
 * the output head's) operand.
 *
 * Groups.  Both norms divide every group of columns by its own root mean square: group g is columns
 * [g * group_cols, (g + 1) * group_cols), width / groups of them true ones and the rest zero.  With one group group_cols
 * is not looked at.
 *
 * Input convolution (single tokens).  With `conv` the operand is h + sum_j conv[j] * h_(t - taps + 1 + j), h the normed row
 * rounded to the element type, its last inputs in conv_state (as tah_conv_rows leaves them), where h is entered. */
typedef struct tah_residual_norm_args {
    const void* y;            /* [rows, y_row_stride], or NULL */
    const float* y_scale;     /* [rows], or NULL: 1 */
    const void* experts;      /* rows of expert outputs, or NULL */
    const int32_t* index;     /* [rows, top] */
    const float* weight;      /* [rows, top] */
    const float* coef;        /* [cols] */
    const float* next_coef;   /* [cols], or NULL */
    float* x;                 /* [rows, cols], updated in place */
    void* xe;                 /* element type [rows, cols], or NULL */
    void* x_packed;           /* bf16 rows form, or NULL */
    void* normed;             /* element type [rows, cols], or NULL */
    void* normed_packed;      /* bf16 rows form, or NULL */
    int64_t y_row_stride, experts_row_stride;
    int32_t rows, width, cols, top, index_scale, index_row, dtype;
    float eps;
    int32_t groups, group_cols;
    const float* conv;        /* [taps, cols], or NULL */
    void* conv_state;         /* element type [nslots, taps, cols] */
    const int32_t *slot, *pos; /* [rows], with conv */
    int32_t taps, nslots;
} tah_residual_norm_args;
int tah_residual_norm(const tah_residual_norm_args* args, tah_stream_t stream);

/* out[r][c] = f(in[r][c]), or for the gates f(in[r][c], in[r][cols + c]), c < cols: gelu (tanh form); silu(g) u; xielu,
 * c0 x^2 + x / 2 above zero and c1 (exp(x) - 1 - x) + x / 2 below; the clamped gate g sigmoid(c1 g) (u + 1) with g =
 * min(g, c0), u = clamp(u, -c0, c0). */
enum { TAH_ROWS_GELU_TANH = 0, TAH_ROWS_SILU_MUL = 1, TAH_ROWS_XIELU = 2, TAH_ROWS_CLAMPED_GATE = 3 };
int tah_activate_rows(const void* in, int64_t in_row_stride, void* out, int64_t out_row_stride, int32_t rows, int32_t cols,
                      int32_t kind, float c0, float c1, int32_t dtype, tah_stream_t stream);

/* Portions' rows h [rows, cols] -> h + causal convolution of h over time, per channel: out[t] = h[t] + sum_j conv[j] *
 * h[t - taps + 1 + j], zeros before a sequence's start.  conv_state element type [nslots, taps, cols]: the last taps - 1
 * inputs of a slot's sequence, token p at p % taps, read for a portion's first rows and brought up to its last ones. */
int tah_conv_rows(const void* h, const float* conv, void* conv_state, const tah_portions* p, void* out, int32_t cols, int32_t taps,
                  int32_t nslots, int32_t dtype, tah_stream_t stream);

/* ---- gated delta rule ---------------------------------------------------------------------------------------- *
 * Per head, with state S [dim, vdim] in float32:  S = g S;  u = beta (v - S^T k);  S = S + k u^T;  o = S^T q, where
 * q, k, v went through a short causal convolution per channel and silu, q and k are unit vectors (q also times
 * dim^-1/2), beta = sigmoid(b), g = exp(-exp(a_log) softplus(a + dt_bias)); the result is
 * o / sqrt(mean(o^2) + eps) * norm * silu(gate). */
typedef struct tah_delta_layer {
    const void* proj;         /* rows of the layer's projections, element type: q [kv_heads * dim] at column q_col, k,
                               * v [heads * vdim], gate [heads * vdim], b [heads], a [heads] */
    int64_t proj_row_stride;
    int32_t q_col, k_col, v_col, gate_col, b_col, a_col;
    const float* conv;        /* [channels, taps], channels = q, k, v one after another; last tap = the current token */
    const float *a_log, *dt_bias; /* [heads] */
    const float* norm;        /* [vdim] */
    void* conv_state;         /* element type [nslots, taps, channels]: inputs of the convolution, token p at p % taps */
    float* state;             /* [nslots, heads, dim, vdim] */
    int32_t heads, kv_heads, dim, vdim, taps, nslots, dtype;
    float eps;
} tah_delta_layer;

/* One token per row: convolution, recurrence, read-out, norm and gate in one launch.  slot, pos int32 [rows];
 * out element type [rows, out_row_stride] (columns heads * vdim .. out_cols are cleared) and / or out_packed, the rows
 * form [32 * out_cols] (rows <= 32). */
int tah_delta_step(const tah_delta_layer* layer, const int32_t* slot, const int32_t* pos, int32_t rows, void* out,
                   int64_t out_row_stride, void* out_packed, int32_t out_cols, tah_stream_t stream);

/* Portions of sequences.  tah_delta_prepare: q, k [T, kv_heads, dim], v [T, heads, vdim], the decay's logarithm and
 * beta [T, heads], all float32, and the convolution's state; row_seq int32 [T]: a row's sequence.
 * tah_delta_scan: the recurrence, o float32 [T, heads, vdim], and the new states; workspace as large as
 * tah_delta_scan_workspace says (0: none), which depends on the sizes and counts alone.
 * tah_delta_finish: norm and gate, out element type [T, out_row_stride]. */
int tah_delta_prepare(const tah_delta_layer* layer, const tah_portions* p, float* q, float* k, float* v, float* log_decay,
                      float* beta, tah_stream_t stream);
int tah_delta_scan(const tah_delta_layer* layer, const tah_portions* p, const float* q, const float* k, const float* v,
                   const float* log_decay, const float* beta, float* o, void* workspace, size_t workspace_bytes, tah_stream_t stream);
size_t tah_delta_scan_workspace(const tah_delta_layer* layer, int32_t nseq, int32_t rows);
int tah_delta_finish(const tah_delta_layer* layer, const float* o, int32_t rows, void* out, int64_t out_row_stride,
                     int32_t out_cols, tah_stream_t stream);

/* ---- latent attention ---------------------------------------------------------------------------------------- *
 * Keys and values are linear in a latent c [rank] per token; a rotated key part [rot_dim] is shared by the heads.
 * What is cached per token is one row [rank_pad + rot_pad]: c, then the rotated part, both zero-padded.  A slot's
 * cache is a ring of `capacity` rows, token p at p % capacity. */
typedef struct tah_latent_layer {
    void* ring;               /* element type [nslots, capacity, rank_pad + rot_pad] */
    int32_t heads, dim_pad, rot_dim, rot_pad, rank, rank_pad, vdim_pad, capacity, nslots, dtype;
    int32_t window;           /* position i sees j with 0 <= i - j < window */
    float scale;
} tah_latent_layer;

/* Rows of projections -> normed latents, rotated key and query parts.  proj: per head [dim_pad | rot_pad] query columns
 * at q_col (rotated in place), and at dkv_col (negative: the layer has none) rank + rot_dim columns.  The new rows go to
 * rows_out [rows, rank_pad + rot_pad] and / or, with slot given, into the ring.  The unrotated query part is also
 * written as the operand of the per-head products: q_packed, rows form per head [heads][32 * dim_pad], or
 * q_rows, element type [heads, rows, dim_pad].  cos, sin float32 [positions, rot_dim / 2]. */
typedef struct tah_latent_prep_args {
    void* proj;
    int64_t proj_row_stride;
    int32_t q_col, dkv_col;
    const float* norm;        /* [rank] */
    const float *cos, *sin;
    const int32_t* pos;       /* [rows] */
    const int32_t* slot;      /* [rows], or NULL */
    void *rows_out, *q_packed, *q_rows;
    int32_t rows, table_rows;
    float eps;
} tah_latent_prep_args;
int tah_latent_prep(const tah_latent_layer* layer, const tah_latent_prep_args* args, tah_stream_t stream);

/* What portions can see, packed: context row cu_k[b] + j of sequence b is position pos0[b] + (cu[b+1] - cu[b]) -
 * (cu_k[b+1] - cu_k[b]) + j, from the ring for positions before the portion, from new_rows (tah_latent_prep's rows_out)
 * for its own; ctx_rows = cu_k[nseq].  Then the last `capacity` new rows of every portion go into the ring. */
int tah_latent_context(const tah_latent_layer* layer, const tah_portions* p, const int32_t* cu_k, int32_t ctx_rows,
                       const void* new_rows, void* ctx, tah_stream_t stream);

/* Attention of portions.  q as tah_latent_prep left it in proj; k [ctx_rows, heads, dim_pad] and v [ctx_rows, heads,
 * vdim_pad] are products of the context's latents (row strides k_row_stride, v_row_stride), ctx gives the rotated key
 * part.  out element type [rows, out_row_stride]: head h at column h * vdim_pad.  max_rows: rows of the longest
 * portion. */
int tah_latent_attend(const tah_latent_layer* layer, const tah_portions* p, const int32_t* cu_k, int32_t max_rows,
                      const void* q, int64_t q_row_stride, const void* k, int64_t k_row_stride, const void* v,
                      int64_t v_row_stride, const void* ctx, void* out, int64_t out_row_stride, tah_stream_t stream);

/* Attention of single tokens straight on the ring: q_latent [heads, rows, rank_pad] is the unrotated query carried
 * over to latent coordinates, q at q_col as above gives the rotated part.  The result, the weighted sum of latents, goes
 * to out_packed, rows form per head [heads][32 * rank_pad], or out_rows [heads, rows, rank_pad].
 * workspace: tah_latent_decode_workspace bytes. */
size_t tah_latent_decode_workspace(const tah_latent_layer* layer, int32_t rows);
int tah_latent_decode(const tah_latent_layer* layer, const int32_t* slot, const int32_t* pos, int32_t rows, const void* q_latent,
                      int64_t q_latent_head_stride, const void* q, int64_t q_row_stride, void* out_packed, void* out_rows,
                      void* workspace, size_t workspace_bytes, tah_stream_t stream);

/* ---- attention in a sliding window with kept first tokens ---------------------------------------------------------- *
 * Position i sees j <= i with i - j < window or j < keep_first.  Query head h reads key/value head h / (heads / kv_heads).
 * What a token caches per key/value head is one row of `row` elements in which the values are columns [0, value_dim) and
 * the keys [row - key_dim, row); the two may overlap, so that keys which are also the values are kept once.  The
 * last rot_pad columns of a key (and of a query, key_dim elements) hold the rotated part, entries 2 i and 2 i + 1 a pair,
 * rot_dim of them and zeros behind; a new row brings the pairs unrotated at column rot_source.  A slot's cache is
 * keep_first rows for the first tokens and a ring: token p at row p (p < keep_first), else keep_first + (p - keep_first)
 * % ring. */
typedef struct tah_window_layer {
    void* cache;              /* element type [nslots, kv_heads, keep_first + ring, row] */
    int32_t heads, kv_heads, row, key_dim, value_dim, rot_dim, rot_pad, rot_source;
    int32_t keep_first, ring, window, nslots, dtype;
    float scale;
} tah_window_layer;
/* Rows of a step: projections with a query head's key_dim columns at q_col + h * key_dim, a key/value head's row at
 * k_col + g * row, and (g_col >= 0) a gate per head: head h's result is multiplied by sigmoid of column g_col + h. */
typedef struct tah_window_rows {
    void* proj;
    int64_t proj_row_stride;
    const float *cos, *sin;   /* float32 [table_rows, rot_dim / 2] */
    const int32_t* pos;       /* [rows] */
    const int32_t* slot;      /* [rows], or NULL */
    int32_t q_col, k_col, g_col, rows, table_rows;
} tah_window_rows;
/* Rotates queries and keys in place; with `slot` the rows also go into their slots' caches. */
int tah_window_prep(const tah_window_layer* layer, const tah_window_rows* rows, tah_stream_t stream);
/* Attention of portions on prepared rows, which are the portions' own keys, and on the cache for the positions before
 * them.  out element type [rows, out_row_stride]: head h at column h * value_dim. */
int tah_window_attend(const tah_window_layer* layer, const tah_portions* p, const tah_window_rows* rows, void* out, int64_t out_row_stride,
                      tah_stream_t stream);
/* The portions' prepared rows into the cache (behind tah_window_attend, which reads what they replace). */
int tah_window_append(const tah_window_layer* layer, const tah_portions* p, const tah_window_rows* rows, tah_stream_t stream);
/* Single tokens: rotation, cache entry and attention.  out element type [rows, out_row_stride] and / or out_packed, the
 * rows form [32 * heads * value_dim] (rows <= 32).  workspace: tah_window_decode_workspace bytes. */
size_t tah_window_decode_workspace(const tah_window_layer* layer, int32_t rows);
int tah_window_decode(const tah_window_layer* layer, const tah_window_rows* rows, void* out, int64_t out_row_stride, void* out_packed,
                      void* workspace, size_t workspace_bytes, tah_stream_t stream);

/* ---- mixture of experts -------------------------------------------------------------------------------------- *
 * tah_moe_route: logits x . router in float32; scores are the logits (TAH_MOE_SOFTMAX) or their sigmoids (TAH_MOE_SIGMOID).
 * The experts form `groups` equal groups of neighbours (1: none); with keep < groups only the `keep` groups with the
 * largest sum of their two largest scores are open.  index: the `top` largest scores of the open experts (the lower index
 * among equals); weight: softmax over the chosen logits, or the chosen scores.  shared_gate = sigmoid(x . gate_w) when
 * gate_w is given.  x [rows, cols] float32, or (x_elem) of the element type; router, gate_w element type. */
enum { TAH_MOE_SOFTMAX = 0, TAH_MOE_SIGMOID = 1 };
typedef struct tah_moe_route_args {
    const void *x, *router, *gate_w;
    int32_t* index;           /* [rows, top] */
    float* weight;            /* [rows, top] */
    float* shared_gate;       /* [rows], or NULL */
    int32_t rows, cols, experts, top, groups, keep, score, x_elem, dtype;
} tah_moe_route_args;
int tah_moe_route(const tah_moe_route_args* args, tah_stream_t stream);
/* Rows sorted by expert, every expert's rows padded to whole tiles of TAH_MOE_TILE: source row of every place (-1:
 * padding), the expert of every tile (-1 past the last) and behind them the number of tiles used, and the place of
 * every (row, choice).  source holds tah_moe_places(rows, top, experts) places, tile_expert a tile for each TAH_MOE_TILE
 * of them and one entry more. */
enum { TAH_MOE_TILE = 128 };
int32_t tah_moe_places(int32_t rows, int32_t top, int32_t experts);
int tah_moe_plan(const int32_t* index, int32_t rows, int32_t top, int32_t experts, int32_t* source, int32_t* tile_expert,
                 int32_t* place, tah_stream_t stream);
/* Product of the sorted rows with their experts' weights.  TAH_LINEAR_GATE_UP: w [experts, 2 n, k] (gate rows, then up
 * rows), x row source[place] (`tiles` without the entry behind them), out = silu(gate) * up [places, n], or with TAH_ACT_CLAMPED_GATE the
 * clamped gate with constants c0, c1; TAH_LINEAR_PLAIN: w [experts, n, k], x row `place`. */
int tah_moe_linear(const void* x, int64_t x_row_stride, const void* w, const int32_t* source, const int32_t* tile_expert,
                   int32_t tiles, int32_t n, int32_t k, int32_t kind, int32_t activation, float c0, float c1, void* out,
                   int64_t out_row_stride, int32_t dtype, tah_stream_t stream);

#ifdef __cplusplus
}
#endif
#endif /* TAH_MIXERS_H */
