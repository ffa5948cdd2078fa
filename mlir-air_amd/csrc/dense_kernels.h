// Internal launch interface between the C ABI of the dense-weight library (dense_capi.hip) and its kernel files.
// dtype: 0 = bf16, 1 = float, of weights and activations (`void *`); residual, norms, router logits are always fp32.
#pragma once

#include <hip/hip_runtime.h>
#include <stddef.h>
#include <stdint.h>

namespace w4a16 {

enum : int { kBf16 = 0, kF32 = 1 };
inline size_t elem_bytes(int dtype) { return dtype == kF32 ? 4 : 2; }

// What a one-token product reads as its input vector.
enum : int {
    kIntakePlain = 0,      // x
    kIntakeResidual = 1,   // res + y / rms(y) * norm_w, also left in res_out (and h_out)
    kIntakeEmbed = 2,      // embed[*token] * scale, also left in res_out (and h_out)
    kIntakeFinal = 3,      // the norm final_w of (res + y / rms(y) * norm_w), or of res without y
    kIntakeNormed = 4,     // the norm final_w of v = embed[*token] * scale, res + y or res; v also left in res_out
};
struct RowIntake {
    int mode = kIntakePlain;
    const void *x = nullptr;
    const float *res = nullptr, *y = nullptr, *norm_w = nullptr, *final_w = nullptr;
    float eps = 0.f;
    int width = 0;         // elements that count in the mean (the rest of K is zero padding)
    float *res_out = nullptr;
    void *h_out = nullptr;
    const void *embed = nullptr;
    const int32_t *token = nullptr;
    float scale = 1.f;
};
// What becomes of the row sums: stored as they are, with silu on rows silu_begin .. silu_end - 1, or (gate != 0) combined in pairs:
// W holds 16 gate rows, 16 up rows, ... and out[N / 2] = gate's activation times up.
enum : int { kGateNone = 0, kGateSilu = 1, kGateGelu = 2 };
struct RowOutput {
    int silu_begin = 0, silu_end = 0, gate = kGateNone;
};
// y[N] = W[N, K] x[K]; out in the element type, or fp32 in out_f32.  keys (4 per workgroup): argmax keys of the
// first n_valid rows.
hipError_t launch_dense_gemv(int dtype, const void *w, const RowIntake &in, void *out, float *out_f32, unsigned long long *keys,
                             int n_valid, int K, int N, hipStream_t stream, const RowOutput &ro = RowOutput());
int dense_gemv_blocks(int K, int N);   // workgroups of that launch; it writes four keys per workgroup
// token[0] = argmax from the keys; position[0] += 1; history[position] = token (each optional)
hipError_t launch_argmax_keys(const unsigned long long *keys, int n, int32_t *token, int32_t *position, int32_t *history,
                              hipStream_t stream);

// Experts of one token or of many.
struct Router {
    const float *logits = nullptr;      // [tokens, ld]
    const float *correction = nullptr;  // [experts]
    int ld = 0, experts = 0, top = 0, groups = 1, keep = 1;
};
constexpr int kMaxExperts = 1024, kMaxTop = 32;
// one token: h[top, ff] = silu(gate x) * (up x) of the chosen experts; ids and weights of the choice are left for the
// second product, y[width] = sum_s weight_s down_s h_s
hipError_t launch_moe_gate_up_gemv(int dtype, const Router &r, const void *x, const void *w_gate_up, void *h, int32_t *ids, float *weights,
                                   int K, int ff, hipStream_t stream);
hipError_t launch_moe_down_gemv(int dtype, const void *h, const void *w_down, const int32_t *ids, const float *weights, float *y, int top,
                                int ff, int N, hipStream_t stream);
// many tokens
hipError_t launch_moe_select(const Router &r, int tokens, int32_t *ids, float *weights, hipStream_t stream);
// entries (token * top + slot) sorted by expert, and the row tiles of `bm` entries that the grouped product runs over:
// tiles[i] = {expert, first sorted entry, entries, 0}, and behind the most tiles that there can be {number of tiles}
int moe_max_tiles(int entries, int experts, int bm);
hipError_t launch_moe_plan(const int32_t *ids, int entries, int experts, int bm, int32_t *order, int32_t *tiles, hipStream_t stream);

// Products over many rows: out[M, N] = A[M, K] W[N, K]^T.
// swiglu, geglu: W holds 16 gate rows, 16 up rows, ...; out is [M, N / 2], silu or the tanh form of gelu of the gate times up
enum : int { kOutElem = 0, kOutF32 = 1, kOutSwiglu = 2, kOutGeglu = 3 };
struct GemmArgs {
    const void *a = nullptr, *w = nullptr;
    void *out = nullptr;
    int M = 0, N = 0, K = 0;
    long lda = 0, ldo = 0;
    int epilogue = kOutElem;
    // grouped (experts): rows are sorted entries, tiles from launch_moe_plan
    const int32_t *tiles = nullptr, *order = nullptr;
    int n_tiles = 0;       // the most tiles (moe_max_tiles)
    int gather = 0;        // > 0: A row of an entry = entry / gather, out row = sorted place; 0: A row = sorted place, out row = entry
    long w_stride = 0;     // elements from one expert's W to the next
    int silu_begin = 0, silu_end = 0;   // columns that silu is applied to (kOutElem, multiples of 16)
};
int dense_gemm_tile_rows(int dtype, int rows, int N, int matrices);   // rows of a tile (what launch_moe_plan gets as bm)
hipError_t launch_dense_gemm(int dtype, const GemmArgs &g, int tile_rows, hipStream_t stream);

// v = embed[tokens] * scale, or res + y, or res; res = v; h (optional) = the norm norm_w of v in the element type
hipError_t launch_add_norm_rows(int dtype, float *res, const float *y, const int32_t *tokens, const void *embed, float scale, const float *norm_w,
                                float eps, int true_width, void *h, int M, int width, hipStream_t stream);
hipError_t launch_embed_rows(int dtype, const int32_t *tokens, const void *embed, float scale, float *res, void *h, int M, int width,
                             hipStream_t stream);
// res += y / rms(y) * norm_w per row; h = res in the element type.  With weights (experts): y is [M * top, width] in the
// element type and the row is sum_s weights[m, s] y[m * top + s]; otherwise y is fp32 [M, width].
hipError_t launch_residual_norm_rows(int dtype, float *res, const void *y, const float *weights, int top, const float *norm_w, float eps,
                                     int true_width, void *h, int M, int width, hipStream_t stream);
// out[i] = norm of res[rows[i]] (rows nullptr: i)
hipError_t launch_norm_rows(int dtype, const float *res, const int32_t *rows, const float *norm_w, float eps, int true_width, void *out, int n,
                            int width, hipStream_t stream);

// Attention of a few rows over a cache, split along the keys: what a cache row is.  Rows of queries are [token][head] within a
// key / value head, [key / value head] outermost; so are the partial results.
struct CacheView {
    int heads = 0, kv_heads = 1;        // query heads of one key / value head, key / value heads
    int q_len = 0, row_len = 0;         // elements that are scored, elements of a cache row
    int v_off = 0, v_cols = 0;          // the part of a row that is summed
    int window = 1 << 30;               // a position sees itself and the window - 1 positions before it
    int ring = 0;                       // rows of the cache that positions go round in (whole blocks of keys), 0: it is as long as the sequence
    long head_stride = 0;               // elements between the matrices of two key / value heads
    float scale = 1.f;
};
// Keys of one split of `n` keys, in whole blocks, and the block that the first visible key lies in: the same for the splits and
// for what merges them.
__host__ __device__ __forceinline__ int keys_per_split(int n, int nsplit, int kb) {
    const int blocks = (n + kb - 1) / kb;
    return (blocks + nsplit - 1) / nsplit * kb;
}
__host__ __device__ __forceinline__ int first_block_key(int pos0, int window, int kb) { return pos0 < window ? 0 : (pos0 - window + 1) / kb * kb; }
int decode_block_keys(int dtype, const CacheView &v);   // keys of a block, 0: no kernel for these sizes
hipError_t launch_cache_decode(int dtype, const CacheView &v, const void *q, const void *cache, int M, const int32_t *pos_dev, int pos, int nsplit,
                               float *part_o, float *part_ml, hipStream_t stream);

// Attention of H query heads over G key / value heads of their own projections (head h: key / value head h / (H / G)), with a norm
// on queries and keys and a window.  A cache row of a key / value head is [key | value]; the heads' matrices follow each other.
struct HeadShape {
    int heads, kv_heads, dim, vdim;     // padded sizes (multiples of 32)
    int true_dim;                       // elements in the mean of the norms
    int window, ring;                   // ring: rows of a head's matrix
    float scale, out_scale;             // of the scores, of the result
};
struct HeadRows {
    const void *proj = nullptr;         // [M, ld]: q of all heads, k and v of all key / value heads from column `off`
    long ld = 0;
    int off = 0;
    const float *q_norm = nullptr, *k_norm = nullptr;
    float eps = 0.f;
    void *cache = nullptr;
    int M = 0;
    const int32_t *pos_dev = nullptr;
    int pos = 0;
};
// normed queries q [kv_heads][M][heads / kv_heads][dim], rows appended to the cache
hipError_t launch_head_prepare(int dtype, const HeadShape &s, const HeadRows &r, void *q, hipStream_t stream);
CacheView head_view(const HeadShape &s);
hipError_t launch_head_merge(int dtype, const HeadShape &s, const HeadRows &r, int nsplit, const float *part_o, const float *part_ml, void *out, long ldo,
                             hipStream_t stream);
hipError_t launch_head_prefill(int dtype, const HeadShape &s, const HeadRows &r, const void *q, void *out, long ldo, hipStream_t stream);
bool head_prefill_supported(int dtype, const HeadShape &s);

// Linear recurrences.  dim is padded to a multiple of 64, vdim of 32.
struct ConvArgs {
    int k_heads, heads, dim, vdim;      // channels: q of k_heads, k of k_heads, v of heads
    int taps;
    long ld;
    int off;                            // column of q in the projections
    const float *w;                     // [taps][channels]
    float *factors;                     // [M][q of k_heads | k of k_heads]: q_scale / |q|, 1 / |k|
    float q_scale, unit_eps;
    int M;
    const int32_t *pos_dev;             // (NULL with more than one token)
    int pos;
};
// act [M, channels]; history [taps, channels]
hipError_t launch_short_conv(int dtype, const ConvArgs &c, const void *proj, void *history, void *act, hipStream_t stream);

struct LinearArgs {
    int k_heads, heads, dim, vdim;
    const void *qkv;                    // [M, ld]: q at q_off, k at k_off (k_heads x dim), v at v_off (heads x vdim)
    long ld;
    int q_off, k_off, v_off;
    const float *log2_decay;            // [heads]: one decay per head, or ...
    const float *z;                     // ... [M, heads x dim]: exp(-exp(a_log) softplus(z + dt_bias)) per channel, and the delta rule
    const float *a_log, *dt_bias;
    const float *factors;               // (delta rule) of ConvArgs
    const void *beta;                   // (delta rule) [M, ld_beta]: sigmoid of it
    long ld_beta;
    float *state;                       // [heads][vdim][dim]
    int M;
    const int32_t *pos_dev;
    int pos;
};
constexpr int kMaxStateDim = 512;
// o [M, heads x vdim]
hipError_t launch_recurrence_steps(int dtype, const LinearArgs &a, float *o, hipStream_t stream);
// long portions by chunks; work: linear_chunk_bytes of device memory
bool linear_chunks_supported(const LinearArgs &a);
size_t linear_chunk_bytes(const LinearArgs &a);
hipError_t launch_linear_chunks(int dtype, const LinearArgs &a, void *work, float *o, hipStream_t stream);

struct GatedNorm {
    const float *o;                     // [M, groups x cols]
    int groups, cols, true_cols;        // a norm runs over the cols of one group
    const float *w;                     // [cols]
    float eps;
    long ld_gate, ld_out;
};
hipError_t launch_gated_norm(int dtype, const GatedNorm &g, const void *gate, void *out, int M, hipStream_t stream);

// Steps of one token that share a launch (r.M, a.M and c.M are 1): attention's preparation and a state step with a decay per head ...
hipError_t launch_head_state_begin(int dtype, const HeadShape &s, const HeadRows &r, void *q, const LinearArgs &a, float *o, hipStream_t stream);
// ... the merge of the keys' splits and the norm and gate of the read-outs (one group) ...
hipError_t launch_head_state_end(int dtype, const HeadShape &s, const HeadRows &r, int nsplit, const float *part_o, const float *part_ml, void *out,
                                 const GatedNorm &g, const void *gate, void *norm_out, hipStream_t stream);
// ... a short convolution and two products out[N] = w[N, K] x[K] with short rows, the first one's result fp32
struct ShortProduct {
    const void *w, *x;
    void *out;
    int K, N;
};
hipError_t launch_conv_products(int dtype, const ConvArgs &c, const void *proj, void *history, void *act, const ShortProduct &a, const ShortProduct &b,
                                hipStream_t stream);

// Latent attention.  Sizes are the padded ones; a cache row is [latent kv_rank | rotated key part rot].
struct LatentShape {
    int heads, dim, rot, vdim, rank;    // padded sizes (dim, rot, vdim multiples of 32, rank of 64)
    int rot_pairs;                      // pairs that are rotated (true rot / 2)
    int true_rank;                      // elements in the mean of the latent's norm
    float scale;
};
struct LatentRows {
    const void *proj = nullptr;         // [M, ld]: q per head [dim | rot], then (with_kv) latent | key part, then the gate
    long ld = 0;
    int kv_off = -1;                    // column of the latent, -1: the layer has none
    int gate_off = 0;
    const float *lut = nullptr;         // [positions, rot_pairs, 2]: cos, sin
    const float *kv_norm = nullptr;
    float eps = 0.f;
    void *cache = nullptr;              // [rows, rank + rot]
    int M = 0;
    const int32_t *pos_dev = nullptr;   // position of the first row, on the device ...
    int pos = 0;                        // ... or here
};
// rotates q in place and appends the cache rows
hipError_t launch_latent_prepare(int dtype, const LatentShape &s, const LatentRows &r, hipStream_t stream);
// appends the cache rows and writes the queries against the latent: qa[M * heads, rank + rot]
hipError_t launch_latent_absorb(int dtype, const LatentShape &s, const LatentRows &r, const void *w_uk, void *qa, hipStream_t stream);
// attention of qa over the cache, split along the keys; then merge, value projection and gate: out[M, ldo]
hipError_t launch_latent_decode(int dtype, const LatentShape &s, const LatentRows &r, const void *qa, int nsplit, float *part_o, float *part_ml,
                                hipStream_t stream);
hipError_t launch_latent_combine(int dtype, const LatentShape &s, const LatentRows &r, int nsplit, const float *part_o, const float *part_ml,
                                 const float *sink, const void *w_uv, void *out, long ldo, hipStream_t stream);
bool latent_decode_supported(int dtype, const LatentShape &s);
// causal attention on per-head keys and values kv[T, ldkv] (keys of all heads, then values of all heads)
hipError_t launch_latent_prefill(int dtype, const LatentShape &s, const LatentRows &r, const void *kv, long ldkv, const float *sink, void *out,
                                 long ldo, hipStream_t stream);
bool latent_prefill_supported(int dtype, const LatentShape &s);

}  // namespace w4a16
