/*
 * dense_lm.h - C ABI of the MI355X (gfx950) kernels for models with dense (bf16 or fp32) weights: one-token and many-row
 * products, latent attention, windowed attention of grouped heads, linear recurrences over a matrix state, a mixture of experts,
 * the row-wise steps between them.
 *
 * One shared library (libdense_lm_hip.so), separate from libw4a16_hip.so so that each can be built alone.  The conventions
 * are those of w4a16.h: all data pointers are DEVICE pointers owned by the caller (the descriptor structs themselves are
 * host memory, read during the call), nothing here allocates device memory, every entry point returns DLM_OK (0) or a
 * negative DLM_ERR_* code, arguments are validated before the first HIP call, `stream` is a hipStream_t passed as void*
 * and launches are asynchronous on it.
 *
 * dtype: DLM_BF16 (weights and activations bf16, sums fp32) or DLM_F32 (everything in true fp32).  The residual stream,
 * norm weights, sinks, router logits and corrections are fp32 in both, and so are recurrent states and all that enters them
 * except projections and short convolutions.
 *
 * Sizes are padded by the caller, with zeros: the input length K of every product to a multiple of 64, its output length
 * to a multiple of 16, a head's dim, rot and vdim to multiples of 32 (a recurrence's dim of 64), the latent's rank to a multiple
 * of 64.  Where the true size matters (the mean of a norm) it is passed beside the padded one.
 */
#ifndef DENSE_LM_H
#define DENSE_LM_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define DLM_OK 0
#define DLM_ERR_NULL (-1)
#define DLM_ERR_SHAPE (-2)
#define DLM_ERR_ALIGN (-4)
#define DLM_ERR_HIP (-6)

#define DLM_BF16 0
#define DLM_F32 1

#define DLM_ABI_VERSION 2

int dlm_abi_version(void);
const char *dlm_strerror(int code);
const char *dlm_last_hip_error(void);

/* The input vector of a one-token product.  mode 0: x.  1: res + y / rms(y) * norm_w, also left in res_out (fp32) and, if
 * given, h_out.  2: embed[*token] * scale, left in the same places.  3: the norm final_w of (res + y / rms(y) * norm_w), or
 * of res if y is NULL.  4: the norm final_w of v = embed[*token] * scale (embed given), res + y or res; v is left in res_out if
 * given.  All vectors have K elements of which `width` count in the means. */
typedef struct {
    int32_t mode, width;
    float eps, scale;
    const void *x;
    const float *res, *y, *norm_w, *final_w;
    float *res_out;
    void *h_out;
    const void *embed;
    const int32_t *token;
} dlm_intake;

/* y[N] = W[N, K] x[K]: `out` in the element type or `out_f32` (exactly one of them).  keys (optional,
 * dlm_gemv_keys(K, N) words): for dlm_argmax over the first n_valid rows. */
int dlm_gemv_keys(int K, int N);
int dlm_gemv(int dtype, const void *w, const dlm_intake *in, void *out, float *out_f32, uint64_t *keys, int n_valid, int K, int N,
             void *stream);
/* The same with something done to the sums: silu on rows silu_begin .. silu_end - 1, or gate 1 (silu) / 2 (tanh form of gelu):
 * W holds 16 gate rows, 16 up rows, ... and out[N / 2] = activation(gate) * up (intakes 0 and 4). */
typedef struct {
    int32_t silu_begin, silu_end, gate;
} dlm_row_output;
int dlm_gemv_act(int dtype, const void *w, const dlm_intake *in, const dlm_row_output *ro, void *out, int K, int N, void *stream);
/* token[0] = row with the largest value (lowest row on ties); position[0] += 1; history[position] = token.  Each optional. */
int dlm_argmax(const uint64_t *keys, int n_keys, int32_t *token, int32_t *position, int32_t *history, void *stream);

/* Grouped sigmoid router: scores sigmoid(logits), choice by score + correction among the `keep` best of `groups` equal groups
 * of neighbours (a group counts as the sum of its two largest choice scores), weights = scores of the `top` chosen. */
typedef struct {
    const float *logits;      /* [tokens, ld] */
    const float *correction;  /* [experts] */
    int32_t ld, experts, top, groups, keep;
} dlm_router;
/* One token.  w_gate_up [experts, 2 ff, K]: 16 gate rows, 16 up rows, 16 gate rows, ...; h[top, ff], ids[top],
 * weights[top] are written and read by the second call: y[N] = sum_s weights[s] * w_down[ids[s]] h[s], w_down
 * [experts, N, ff]. */
int dlm_moe_gate_up_gemv(int dtype, const dlm_router *r, const void *x, const void *w_gate_up, void *h, int32_t *ids, float *weights,
                         int K, int ff, void *stream);
int dlm_moe_down_gemv(int dtype, const void *h, const void *w_down, const int32_t *ids, const float *weights, float *y, int top,
                      int experts, int ff, int N, void *stream);
/* Many tokens: ids, weights [tokens, top]; then the entries token * top + slot sorted by expert (order[tokens * top]) and
 * their row tiles (int32 [dlm_moe_max_tiles(..) + 1, 4]; the last row holds the number of tiles in use). */
int dlm_moe_select(const dlm_router *r, int tokens, int32_t *ids, float *weights, void *stream);
int dlm_moe_max_tiles(int entries, int experts, int tile_rows);
int dlm_moe_plan(const int32_t *ids, int entries, int experts, int tile_rows, int32_t *order, int32_t *tiles, void *stream);

/* out[M, N] = A[M, K] W[N, K]^T.  epilogue 0: element type, with silu on columns silu_begin .. silu_end - 1 (multiples of 16, not
 * grouped), 1: fp32, 2: SwiGLU of interleaved gate / up rows (out [M, N / 2]), 3: the same with the tanh form of gelu (not grouped).  Grouped: tiles != NULL, W [experts, ..] with w_stride elements per expert, M = entries; gather > 0: the A
 * row of an entry is entry / gather and out rows are sorted places; gather 0: A rows are sorted places, out rows entries. */
typedef struct {
    const void *a, *w;
    void *out;
    int64_t lda, ldo, w_stride;
    const int32_t *tiles, *order;
    int32_t M, N, K, epilogue, n_tiles, gather, tile_rows;   /* tile_rows: dlm_gemm_tile_rows, or 32, 128, 256 */
    int32_t silu_begin, silu_end;
} dlm_gemm_args;
/* Rows of A per tile for `rows` rows (experts: the mean number) with each of `matrices` matrices of N rows. */
int dlm_gemm_tile_rows(int dtype, int rows, int N, int matrices);
int dlm_gemm(int dtype, const dlm_gemm_args *g, void *stream);

int dlm_embed_rows(int dtype, const int32_t *tokens, const void *embed, float scale, float *res, void *h, int M, int width, void *stream);
/* res += y / rms(y) * norm_w; h (optional) = res in the element type.  weights NULL: y fp32 [M, width]; otherwise y in the
 * element type [M * top, width], summed with weights[M, top] first. */
int dlm_residual_norm_rows(int dtype, float *res, const void *y, const float *weights, int top, const float *norm_w, float eps,
                           int true_width, void *h, int M, int width, void *stream);
/* v = embed[tokens] * scale (tokens given), res + y (y given) or res; res = v, h (optional) = v / rms(v) * norm_w in the element type */
int dlm_add_norm_rows(int dtype, float *res, const float *y, const int32_t *tokens, const void *embed, float scale, const float *norm_w, float eps,
                      int true_width, void *h, int M, int width, void *stream);
/* out[i] = res[rows[i]] / rms * norm_w in the element type (rows NULL: i) */
int dlm_norm_rows(int dtype, const float *res, const int32_t *rows, const float *norm_w, float eps, int true_width, void *out, int n,
                  int width, void *stream);

/* Latent attention.  A cache row is [latent (rank) | rotated key part (rot)]. */
typedef struct {
    int32_t heads, dim, rot, vdim, rank; /* padded */
    int32_t rot_pairs, true_rank;
    float scale;
} dlm_latent_shape;
typedef struct {
    const void *proj;        /* [M, ld]: q per head [dim | rot], latent | key part at kv_off (-1: none), gate at gate_off */
    const float *lut;        /* [positions, rot_pairs, 2]: cos, sin */
    const float *kv_norm;    /* [rank] */
    void *cache;             /* rows of rank + rot */
    const int32_t *pos_dev;  /* position of the first row on the device, or NULL and `pos` */
    int64_t ld;
    int32_t kv_off, gate_off, M, pos;
    float eps;
} dlm_latent_rows;
int dlm_latent_decode_supported(int dtype, const dlm_latent_shape *s);
int dlm_latent_prefill_supported(int dtype, const dlm_latent_shape *s);
/* Long portions: rotate q in place, append the cache rows; then causal attention on kv [pos + M, ldkv] (keys of all heads,
 * values of all heads), gated, out [M, ldo].  (pos_dev must be NULL in dlm_latent_prefill.) */
int dlm_latent_prepare(int dtype, const dlm_latent_shape *s, const dlm_latent_rows *r, void *stream);
int dlm_latent_prefill(int dtype, const dlm_latent_shape *s, const dlm_latent_rows *r, const void *kv, int64_t ldkv, const float *sink,
                       void *out, int64_t ldo, void *stream);
/* One token or short portions: qa [M * heads, rank + rot]; part_o fp32 [M * heads, nsplit, rank], part_ml
 * [M * heads, nsplit, 2]; nsplit <= 256. */
int dlm_latent_absorb(int dtype, const dlm_latent_shape *s, const dlm_latent_rows *r, const void *w_uk, void *qa, void *stream);
int dlm_latent_decode(int dtype, const dlm_latent_shape *s, const dlm_latent_rows *r, const void *qa, int nsplit, float *part_o,
                      float *part_ml, void *stream);
int dlm_latent_combine(int dtype, const dlm_latent_shape *s, const dlm_latent_rows *r, int nsplit, const float *part_o,
                       const float *part_ml, const float *sink, const void *w_uv, void *out, int64_t ldo, void *stream);

/* Softmax attention of `heads` query heads over kv_heads key / value heads (head h: h / (heads / kv_heads)), queries and keys normed
 * per head, a position seeing itself and the window - 1 before it.  A key / value head's cache is `ring` rows [key | value] of
 * dim + vdim, position p in row p % ring; ring is a multiple of 64 and at least window - 1 + M (or the whole sequence). */
typedef struct {
    int32_t heads, kv_heads, dim, vdim; /* padded */
    int32_t true_dim, window, ring;
    float scale, out_scale;
} dlm_head_shape;
typedef struct {
    const void *proj;        /* [M, ld]: from column off on q (heads x dim), k (kv_heads x dim), v (kv_heads x vdim) */
    const float *q_norm, *k_norm;
    void *cache;             /* [kv_heads, ring, dim + vdim] */
    const int32_t *pos_dev;  /* position of the first row on the device, or NULL and `pos` */
    int64_t ld;
    int32_t off, M, pos;
    float eps;
} dlm_head_rows;
int dlm_head_decode_supported(int dtype, const dlm_head_shape *s);
int dlm_head_prefill_supported(int dtype, const dlm_head_shape *s);
/* Normed queries q [kv_heads, M, heads / kv_heads, dim] and the cache rows; then either the attention of many rows, or of few with
 * the keys split (part_o fp32 [kv_heads * M * heads / kv_heads, nsplit, vdim], part_ml [.., nsplit, 2]; nsplit <= 256) and the merge.
 * out [M, ldo] = out_scale * attention.  (pos_dev must be NULL in dlm_head_prefill.) */
int dlm_head_prepare(int dtype, const dlm_head_shape *s, const dlm_head_rows *r, void *q, void *stream);
int dlm_head_prefill(int dtype, const dlm_head_shape *s, const dlm_head_rows *r, const void *q, void *out, int64_t ldo, void *stream);
int dlm_head_decode(int dtype, const dlm_head_shape *s, const dlm_head_rows *r, const void *q, int nsplit, float *part_o, float *part_ml,
                    void *stream);
int dlm_head_merge(int dtype, const dlm_head_shape *s, const dlm_head_rows *r, int nsplit, const float *part_o, const float *part_ml, void *out,
                   int64_t ldo, void *stream);

/* Causal convolution over time per channel, then silu: act [M, C], C = 2 k_heads dim + heads vdim channels (q, k, v), w [taps, C]
 * (the last row meets the current token).  history [taps, C] holds earlier rows by position % taps (rows in front of the sequence
 * count as zeros) and is brought forward.  factors [M, 2 k_heads]: q_scale / |q| per head, then 1 / |k|, |x| = sqrt(sum x^2 +
 * unit_eps). */
typedef struct {
    const void *proj;        /* [M, ld], the channels from column off on */
    const float *w;
    void *history;
    float *factors;
    const int32_t *pos_dev;  /* (one token only) */
    int64_t ld;
    int32_t k_heads, heads, dim, vdim, taps, off, M, pos;
    float q_scale, unit_eps;
} dlm_short_conv_args;
int dlm_short_conv(int dtype, const dlm_short_conv_args *c, void *act, void *stream);

/* S <- g S; u = v, or u = beta (v - S^T k); S <- S + k u^T; o = S^T q per head; head h uses q / k head h / (heads / k_heads).  The
 * state is fp32 [heads, vdim, dim] and is not read at position 0.  log2_decay given: g = 2^log2_decay per head, u = v.  z given
 * (fp32 [M, heads dim]): g = exp(-exp(a_log) softplus(z + dt_bias)) per channel, the delta rule, q and k times their factors,
 * beta = sigmoid of its logit. */
typedef struct {
    const void *qkv;         /* [M, ld]: q at q_off, k at k_off, v at v_off */
    const float *log2_decay, *z, *a_log, *dt_bias, *factors;
    const void *beta;        /* [M, ld_beta] */
    float *state;
    const int32_t *pos_dev;
    int64_t ld, ld_beta;
    int32_t k_heads, heads, dim, vdim, q_off, k_off, v_off, M, pos;
} dlm_recurrence_args;
/* o fp32 [M, heads vdim].  _steps: token by token; _chunks: 64 tokens at a time, work of dlm_recurrence_chunk_bytes (0: no kernel for
 * this size). */
int dlm_recurrence_steps(int dtype, const dlm_recurrence_args *a, float *o, void *stream);
size_t dlm_recurrence_chunk_bytes(const dlm_recurrence_args *a);
int dlm_recurrence_chunks(int dtype, const dlm_recurrence_args *a, void *work, float *o, void *stream);
/* out[m, c] = o / rms * w * sigmoid(gate), the mean running over true_cols of the `cols` columns of a group; o [M, groups cols],
 * w [cols] */
int dlm_gated_norm(int dtype, const float *o, const float *w, const void *gate, int64_t ld_gate, void *out, int64_t ld_out, int M, int groups, int cols,
                   int true_cols, float eps, void *stream);

/* Steps of one token (M = 1) that do not wait for each other in one launch.  _begin: dlm_head_prepare and dlm_recurrence_steps (a decay
 * per head); _end: dlm_head_merge into out and the norm and gate (dlm_gated_norm with one group) into norm_out; dlm_conv_products:
 * dlm_short_conv and out_a[Na] (fp32) = w_a[Na, Ka] x_a, out_b[Nb] (element type) = w_b[Nb, Kb] x_b (K multiples of 64, N of 16). */
int dlm_head_state_begin(int dtype, const dlm_head_shape *s, const dlm_head_rows *r, void *q, const dlm_recurrence_args *a, float *o, void *stream);
int dlm_head_state_end(int dtype, const dlm_head_shape *s, const dlm_head_rows *r, int nsplit, const float *part_o, const float *part_ml, void *out,
                       const float *o, const float *w, const void *gate, int cols, int true_cols, float eps, void *norm_out, void *stream);
typedef struct {
    const void *w, *x;
    void *out;
    int32_t K, N;
} dlm_short_product;
int dlm_conv_products(int dtype, const dlm_short_conv_args *c, void *act, const dlm_short_product *a, const dlm_short_product *b, void *stream);

#ifdef __cplusplus
}
#endif
#endif /* DENSE_LM_H */
