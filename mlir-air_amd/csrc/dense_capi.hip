// C ABI of the dense-weight library (include/dense_lm.h): argument checks, then the launches of dense_kernels.h.
#include "../../include/dense_lm.h"

#include <string>

#include "dense_kernels.h"

using namespace w4a16;

namespace {

thread_local std::string g_error;

int done(hipError_t e) {
    if (e == hipSuccess) return DLM_OK;
    g_error = hipGetErrorString(e);
    return DLM_ERR_HIP;
}
bool odd(const void *p) { return reinterpret_cast<uintptr_t>(p) & 15; }
bool bad_type(int dtype) { return dtype != kBf16 && dtype != kF32; }
hipStream_t hs(void *s) { return static_cast<hipStream_t>(s); }
constexpr int kMaxLength = 16384;   // input length of a product that is staged in LDS
constexpr int kMaxWidth = 15360;    // of a row whose sum is kept in LDS

int check_router(const dlm_router *r) {
    if (!r || !r->logits || !r->correction) return DLM_ERR_NULL;
    if (r->experts <= 0 || r->experts > kMaxExperts || r->top <= 0 || r->top > kMaxTop || r->groups <= 0 || r->experts % r->groups || r->keep <= 0 ||
        r->keep > r->groups || r->top > r->keep * (r->experts / r->groups) || r->ld < r->experts)
        return DLM_ERR_SHAPE;
    return DLM_OK;
}
Router router_of(const dlm_router *r) { return {r->logits, r->correction, r->ld, r->experts, r->top, r->groups, r->keep}; }

int check_latent(int dtype, const dlm_latent_shape *s, const dlm_latent_rows *r) {
    if (!s || !r || !r->proj || !r->lut || !r->cache) return DLM_ERR_NULL;
    if (bad_type(dtype) || s->heads <= 0 || s->dim <= 0 || s->dim % 32 || s->rot <= 0 || s->rot % 32 || s->vdim <= 0 || s->vdim % 32 || s->rank <= 0 ||
        s->rank % 64 || s->rot_pairs <= 0 || 2 * s->rot_pairs > s->rot || s->true_rank <= 0 || s->true_rank > s->rank || !(s->scale > 0.f) || r->M <= 0 ||
        r->M > 65535 || r->pos < 0 || r->ld % 8 || r->gate_off % 8 || (r->kv_off >= 0 && r->kv_off % 8))
        return DLM_ERR_SHAPE;
    if (r->kv_off >= 0 && !r->kv_norm) return DLM_ERR_NULL;
    if (odd(r->proj) || odd(r->cache)) return DLM_ERR_ALIGN;
    return DLM_OK;
}
LatentShape shape_of(const dlm_latent_shape *s) { return {s->heads, s->dim, s->rot, s->vdim, s->rank, s->rot_pairs, s->true_rank, s->scale}; }
LatentRows rows_of(const dlm_latent_rows *r) {
    return {r->proj, (long)r->ld, r->kv_off, r->gate_off, r->lut, r->kv_norm, r->eps, r->cache, r->M, r->pos_dev, r->pos};
}

int check_head(int dtype, const dlm_head_shape *s, const dlm_head_rows *r) {
    if (!s || !r || !r->proj || !r->cache || !r->q_norm || !r->k_norm) return DLM_ERR_NULL;
    if (bad_type(dtype) || s->heads <= 0 || s->kv_heads <= 0 || s->heads % s->kv_heads || s->dim <= 0 || s->dim % 32 || s->vdim <= 0 || s->vdim % 32 ||
        s->true_dim <= 0 || s->true_dim > s->dim || s->window <= 0 || s->ring <= 0 || s->ring % 64 || !(s->scale > 0.f) || r->M <= 0 || r->M > 65535 || r->pos < 0 ||
        r->ld % 8 || r->off < 0 || r->off % 8 || !(r->eps >= 0.f) || r->M > s->ring)
        return DLM_ERR_SHAPE;
    // keys that are still seen must not share a row with new ones
    if (!r->pos_dev && (int64_t)r->pos + r->M > s->ring && (int64_t)s->window - 1 + r->M > s->ring) return DLM_ERR_SHAPE;
    if (odd(r->proj) || odd(r->cache) || odd(r->q_norm) || odd(r->k_norm)) return DLM_ERR_ALIGN;
    return DLM_OK;
}
HeadShape head_of(const dlm_head_shape *s) {
    return {s->heads, s->kv_heads, s->dim, s->vdim, s->true_dim, s->window, s->ring, s->scale, s->out_scale};
}
HeadRows head_rows_of(const dlm_head_rows *r) {
    return {r->proj, (long)r->ld, r->off, r->q_norm, r->k_norm, r->eps, r->cache, r->M, r->pos_dev, r->pos};
}

int check_recurrence(int dtype, const dlm_recurrence_args *a) {
    if (!a || !a->qkv || !a->state || (!a->log2_decay) == (!a->z)) return DLM_ERR_NULL;
    if (a->z && (!a->a_log || !a->dt_bias || !a->factors || !a->beta)) return DLM_ERR_NULL;
    if (bad_type(dtype) || a->heads <= 0 || a->k_heads <= 0 || a->heads % a->k_heads || a->heads > 65535 || a->dim <= 0 || a->dim % 64 || a->dim > kMaxStateDim ||
        a->vdim <= 0 || a->vdim % 32 || a->M <= 0 || a->pos < 0 || a->ld % 8 || a->q_off < 0 || a->q_off % 8 || a->k_off < 0 || a->k_off % 8 || a->v_off < 0 ||
        a->v_off % 8)
        return DLM_ERR_SHAPE;
    if (odd(a->qkv) || odd(a->state) || odd(a->z) || odd(a->dt_bias)) return DLM_ERR_ALIGN;
    return DLM_OK;
}
int check_conv(int dtype, const dlm_short_conv_args *c, const void *act) {
    if (!c || !c->proj || !c->w || !c->history || !c->factors || !act) return DLM_ERR_NULL;
    if (bad_type(dtype) || c->k_heads <= 0 || c->heads <= 0 || c->dim <= 0 || c->dim % 8 || c->vdim <= 0 || c->vdim % 8 || c->taps <= 0 || c->M <= 0 ||
        c->M > 65535 * 4 || c->pos < 0 || c->ld % 8 || c->off < 0 || c->off % 8 || c->taps > 65535 || (c->pos_dev && c->M > 1) || !(c->unit_eps >= 0.f))
        return DLM_ERR_SHAPE;
    if (odd(c->proj) || odd(c->w) || odd(c->history) || odd(act)) return DLM_ERR_ALIGN;
    return DLM_OK;
}
ConvArgs conv_of(const dlm_short_conv_args *c) {
    return {c->k_heads, c->heads, c->dim, c->vdim, c->taps, (long)c->ld, c->off, c->w, c->factors, c->q_scale, c->unit_eps, c->M, c->pos_dev, c->pos};
}
LinearArgs linear_of(const dlm_recurrence_args *a) {
    LinearArgs l;
    l.k_heads = a->k_heads;
    l.heads = a->heads;
    l.dim = a->dim;
    l.vdim = a->vdim;
    l.qkv = a->qkv;
    l.ld = a->ld;
    l.q_off = a->q_off;
    l.k_off = a->k_off;
    l.v_off = a->v_off;
    l.log2_decay = a->log2_decay;
    l.z = a->z;
    l.a_log = a->a_log;
    l.dt_bias = a->dt_bias;
    l.factors = a->factors;
    l.beta = a->beta;
    l.ld_beta = a->ld_beta;
    l.state = a->state;
    l.M = a->M;
    l.pos_dev = a->pos_dev;
    l.pos = a->pos;
    return l;
}

// Fills the kernel's description of a one-token product's input.
int take_intake(int dtype, const dlm_intake *in, int K, RowIntake &r) {
    if (bad_type(dtype) || K <= 0 || K % 64 || K > kMaxLength * (dtype == kF32 ? 1 : 2)) return DLM_ERR_SHAPE;
    switch (in->mode) {
        case kIntakePlain:
            if (!in->x) return DLM_ERR_NULL;
            break;
        case kIntakeResidual:
            if (!in->res || !in->y || !in->norm_w) return DLM_ERR_NULL;
            break;
        case kIntakeEmbed:
            if (!in->embed || !in->token || !in->res_out) return DLM_ERR_NULL;
            break;
        case kIntakeFinal:
            if (!in->res || !in->final_w || (in->y && !in->norm_w)) return DLM_ERR_NULL;
            break;
        case kIntakeNormed:
            if (!in->final_w || (in->embed ? !in->token : !in->res)) return DLM_ERR_NULL;
            break;
        default: return DLM_ERR_SHAPE;
    }
    if (in->mode != kIntakePlain && (in->width <= 0 || in->width > K || !(in->eps >= 0.f))) return DLM_ERR_SHAPE;
    for (const void *q : {in->x, (const void *)in->res, (const void *)in->y, (const void *)in->norm_w, (const void *)in->final_w, (const void *)in->res_out,
                          (const void *)in->h_out, in->embed})
        if (odd(q)) return DLM_ERR_ALIGN;
    r.mode = in->mode;
    r.x = in->x;
    r.res = in->res;
    r.y = in->y;
    r.norm_w = in->norm_w;
    r.final_w = in->final_w;
    r.eps = in->eps;
    r.width = in->width;
    r.res_out = in->res_out;
    r.h_out = in->h_out;
    r.embed = in->embed;
    r.token = in->token;
    r.scale = in->scale;
    return DLM_OK;
}

}  // namespace

extern "C" {

int dlm_abi_version(void) { return DLM_ABI_VERSION; }

const char *dlm_strerror(int code) {
    switch (code) {
        case DLM_OK: return "ok";
        case DLM_ERR_NULL: return "required pointer is NULL";
        case DLM_ERR_SHAPE: return "unsupported size";
        case DLM_ERR_ALIGN: return "pointer is not 16-byte aligned";
        case DLM_ERR_HIP: return "HIP call failed";
        default: return "unknown error";
    }
}

const char *dlm_last_hip_error(void) { return g_error.c_str(); }

int dlm_gemv_keys(int K, int N) { return K > 0 && N > 0 ? 4 * dense_gemv_blocks(K, N) : 0; }

int dlm_gemv(int dtype, const void *w, const dlm_intake *in, void *out, float *out_f32, uint64_t *keys, int n_valid, int K, int N, void *stream) {
    if (!w || !in || (!out) == (!out_f32)) return DLM_ERR_NULL;
    if (N <= 0 || n_valid < 0 || n_valid > N) return DLM_ERR_SHAPE;
    RowIntake r;
    const int c = take_intake(dtype, in, K, r);
    if (c) return c;
    if (odd(w) || odd(out) || odd(out_f32)) return DLM_ERR_ALIGN;
    return done(launch_dense_gemv(dtype, w, r, out, out_f32, reinterpret_cast<unsigned long long *>(keys), n_valid, K, N, hs(stream)));
}

int dlm_gemv_act(int dtype, const void *w, const dlm_intake *in, const dlm_row_output *ro, void *out, int K, int N, void *stream) {
    if (!w || !in || !ro || !out) return DLM_ERR_NULL;
    if (N <= 0 || ro->gate < kGateNone || ro->gate > kGateGelu) return DLM_ERR_SHAPE;
    if (ro->gate && (N % 32 || (in->mode != kIntakePlain && in->mode != kIntakeNormed) || ro->silu_begin < ro->silu_end)) return DLM_ERR_SHAPE;
    RowIntake r;
    const int c = take_intake(dtype, in, K, r);
    if (c) return c;
    if (odd(w) || odd(out)) return DLM_ERR_ALIGN;
    return done(launch_dense_gemv(dtype, w, r, out, nullptr, nullptr, 0, K, N, hs(stream), RowOutput{ro->silu_begin, ro->silu_end, ro->gate}));
}

int dlm_argmax(const uint64_t *keys, int n_keys, int32_t *token, int32_t *position, int32_t *history, void *stream) {
    if (!keys || (history && !position)) return DLM_ERR_NULL;
    if (n_keys <= 0) return DLM_ERR_SHAPE;
    return done(launch_argmax_keys(reinterpret_cast<const unsigned long long *>(keys), n_keys, token, position, history, hs(stream)));
}

int dlm_moe_gate_up_gemv(int dtype, const dlm_router *r, const void *x, const void *w_gate_up, void *h, int32_t *ids, float *weights, int K, int ff,
                         void *stream) {
    const int c = check_router(r);
    if (c) return c;
    if (!x || !w_gate_up || !h || !ids || !weights) return DLM_ERR_NULL;
    if (bad_type(dtype) || K <= 0 || K % 64 || K > kMaxLength || ff <= 0 || ff % 64) return DLM_ERR_SHAPE;
    if (odd(x) || odd(w_gate_up) || odd(h)) return DLM_ERR_ALIGN;
    return done(launch_moe_gate_up_gemv(dtype, router_of(r), x, w_gate_up, h, ids, weights, K, ff, hs(stream)));
}

int dlm_moe_down_gemv(int dtype, const void *h, const void *w_down, const int32_t *ids, const float *weights, float *y, int top, int experts, int ff, int N,
                      void *stream) {
    if (!h || !w_down || !ids || !weights || !y) return DLM_ERR_NULL;
    if (bad_type(dtype) || top <= 0 || top > kMaxTop || experts <= 0 || ff <= 0 || ff % 64 || N <= 0 ||
        (size_t)top * ((ff + 511) / 512 * 512) * elem_bytes(dtype) > 128 * 1024)
        return DLM_ERR_SHAPE;
    if (odd(h) || odd(w_down)) return DLM_ERR_ALIGN;
    return done(launch_moe_down_gemv(dtype, h, w_down, ids, weights, y, top, ff, N, hs(stream)));
}

int dlm_moe_select(const dlm_router *r, int tokens, int32_t *ids, float *weights, void *stream) {
    const int c = check_router(r);
    if (c) return c;
    if (!ids || !weights) return DLM_ERR_NULL;
    if (tokens <= 0) return DLM_ERR_SHAPE;
    return done(launch_moe_select(router_of(r), tokens, ids, weights, hs(stream)));
}

int dlm_moe_max_tiles(int entries, int experts, int tile_rows) {
    return entries > 0 && experts > 0 && tile_rows > 0 ? moe_max_tiles(entries, experts, tile_rows) : 0;
}

int dlm_moe_plan(const int32_t *ids, int entries, int experts, int tile_rows, int32_t *order, int32_t *tiles, void *stream) {
    if (!ids || !order || !tiles) return DLM_ERR_NULL;
    if (entries <= 0 || experts <= 0 || experts > kMaxExperts || tile_rows <= 0) return DLM_ERR_SHAPE;
    return done(launch_moe_plan(ids, entries, experts, tile_rows, order, tiles, hs(stream)));
}

int dlm_gemm_tile_rows(int dtype, int rows, int N, int matrices) { return dense_gemm_tile_rows(dtype, rows, N, matrices); }

int dlm_gemm(int dtype, const dlm_gemm_args *g, void *stream) {
    if (!g || !g->a || !g->w || !g->out) return DLM_ERR_NULL;
    if (bad_type(dtype) || g->M <= 0 || g->N <= 0 || g->N % 16 || g->K <= 0 || g->K % 64 || g->lda < g->K || g->lda % 8 || g->ldo % 8) return DLM_ERR_SHAPE;
    if (g->tile_rows != 32 && g->tile_rows != 128 && g->tile_rows != 256) return DLM_ERR_SHAPE;
    if (g->tiles) {
        if (!g->order) return DLM_ERR_NULL;
        if (g->n_tiles <= 0 || g->gather < 0 || g->epilogue == kOutF32 || g->epilogue == kOutGeglu || g->silu_begin < g->silu_end || g->w_stride < (int64_t)g->N * g->K) return DLM_ERR_SHAPE;
    }
    const bool paired = g->epilogue == kOutSwiglu || g->epilogue == kOutGeglu;
    if (paired && g->N % 32) return DLM_ERR_SHAPE;
    if (g->silu_begin < g->silu_end && (g->epilogue != kOutElem || g->silu_begin % 16 || g->silu_end % 16)) return DLM_ERR_SHAPE;
    if (g->epilogue < 0 || g->epilogue > kOutGeglu || g->ldo < (paired ? g->N / 2 : g->N)) return DLM_ERR_SHAPE;
    if (odd(g->a) || odd(g->w) || odd(g->out)) return DLM_ERR_ALIGN;
    GemmArgs a;
    a.a = g->a;
    a.w = g->w;
    a.out = g->out;
    a.M = g->M;
    a.N = g->N;
    a.K = g->K;
    a.lda = g->lda;
    a.ldo = g->ldo;
    a.epilogue = g->epilogue;
    a.tiles = g->tiles;
    a.order = g->order;
    a.n_tiles = g->n_tiles;
    a.gather = g->gather;
    a.w_stride = g->w_stride;
    a.silu_begin = g->silu_begin;
    a.silu_end = g->silu_end;
    return done(launch_dense_gemm(dtype, a, g->tile_rows, hs(stream)));
}

int dlm_embed_rows(int dtype, const int32_t *tokens, const void *embed, float scale, float *res, void *h, int M, int width, void *stream) {
    if (!tokens || !embed || !res || !h) return DLM_ERR_NULL;
    if (bad_type(dtype) || M <= 0 || width <= 0 || width % 64) return DLM_ERR_SHAPE;
    if (odd(embed) || odd(res) || odd(h)) return DLM_ERR_ALIGN;
    return done(launch_embed_rows(dtype, tokens, embed, scale, res, h, M, width, hs(stream)));
}

int dlm_residual_norm_rows(int dtype, float *res, const void *y, const float *weights, int top, const float *norm_w, float eps, int true_width, void *h,
                           int M, int width, void *stream) {
    if (!res || !y || !norm_w) return DLM_ERR_NULL;
    if (bad_type(dtype) || M <= 0 || width <= 0 || width % 64 || width > kMaxWidth || true_width <= 0 || true_width > width || !(eps >= 0.f) ||
        (weights && top <= 0))
        return DLM_ERR_SHAPE;
    if (odd(res) || odd(y) || odd(norm_w) || odd(h)) return DLM_ERR_ALIGN;
    return done(launch_residual_norm_rows(dtype, res, y, weights, top, norm_w, eps, true_width, h, M, width, hs(stream)));
}

int dlm_norm_rows(int dtype, const float *res, const int32_t *rows, const float *norm_w, float eps, int true_width, void *out, int n, int width,
                  void *stream) {
    if (!res || !norm_w || !out) return DLM_ERR_NULL;
    if (bad_type(dtype) || n <= 0 || width <= 0 || width % 64 || true_width <= 0 || true_width > width || !(eps >= 0.f)) return DLM_ERR_SHAPE;
    if (odd(res) || odd(norm_w) || odd(out)) return DLM_ERR_ALIGN;
    return done(launch_norm_rows(dtype, res, rows, norm_w, eps, true_width, out, n, width, hs(stream)));
}

int dlm_add_norm_rows(int dtype, float *res, const float *y, const int32_t *tokens, const void *embed, float scale, const float *norm_w, float eps,
                      int true_width, void *h, int M, int width, void *stream) {
    if (!res || (tokens && !embed) || (h && !norm_w)) return DLM_ERR_NULL;
    if (bad_type(dtype) || M <= 0 || width <= 0 || width % 64 || width > kMaxWidth || true_width <= 0 || true_width > width || !(eps >= 0.f) || (tokens && y))
        return DLM_ERR_SHAPE;
    if (odd(res) || odd(y) || odd(embed) || odd(norm_w) || odd(h)) return DLM_ERR_ALIGN;
    return done(launch_add_norm_rows(dtype, res, y, tokens, embed, scale, norm_w, eps, true_width, h, M, width, hs(stream)));
}

int dlm_head_decode_supported(int dtype, const dlm_head_shape *s) {
    return s && !bad_type(dtype) && s->kv_heads > 0 && decode_block_keys(dtype, head_view(head_of(s))) != 0;
}
int dlm_head_prefill_supported(int dtype, const dlm_head_shape *s) { return s && !bad_type(dtype) && head_prefill_supported(dtype, head_of(s)); }

int dlm_head_prepare(int dtype, const dlm_head_shape *s, const dlm_head_rows *r, void *q, void *stream) {
    const int c = check_head(dtype, s, r);
    if (c) return c;
    if (!q) return DLM_ERR_NULL;
    if (odd(q)) return DLM_ERR_ALIGN;
    return done(launch_head_prepare(dtype, head_of(s), head_rows_of(r), q, hs(stream)));
}

int dlm_head_prefill(int dtype, const dlm_head_shape *s, const dlm_head_rows *r, const void *q, void *out, int64_t ldo, void *stream) {
    const int c = check_head(dtype, s, r);
    if (c) return c;
    if (!q || !out) return DLM_ERR_NULL;
    if (r->pos_dev || !head_prefill_supported(dtype, head_of(s)) || ldo % 8 || ldo < (int64_t)s->heads * s->vdim) return DLM_ERR_SHAPE;
    if (odd(q) || odd(out)) return DLM_ERR_ALIGN;
    return done(launch_head_prefill(dtype, head_of(s), head_rows_of(r), q, out, ldo, hs(stream)));
}

int dlm_head_decode(int dtype, const dlm_head_shape *s, const dlm_head_rows *r, const void *q, int nsplit, float *part_o, float *part_ml, void *stream) {
    const int c = check_head(dtype, s, r);
    if (c) return c;
    if (!q || !part_o || !part_ml) return DLM_ERR_NULL;
    const CacheView v = head_view(head_of(s));
    if (nsplit <= 0 || nsplit > 256 || !decode_block_keys(dtype, v)) return DLM_ERR_SHAPE;
    if (odd(q) || odd(part_o)) return DLM_ERR_ALIGN;
    return done(launch_cache_decode(dtype, v, q, r->cache, r->M, r->pos_dev, r->pos, nsplit, part_o, part_ml, hs(stream)));
}

int dlm_head_merge(int dtype, const dlm_head_shape *s, const dlm_head_rows *r, int nsplit, const float *part_o, const float *part_ml, void *out, int64_t ldo,
                   void *stream) {
    const int c = check_head(dtype, s, r);
    if (c) return c;
    if (!part_o || !part_ml || !out) return DLM_ERR_NULL;
    if (nsplit <= 0 || nsplit > 256 || !decode_block_keys(dtype, head_view(head_of(s))) || ldo % 8 || ldo < (int64_t)s->heads * s->vdim) return DLM_ERR_SHAPE;
    if (odd(part_o) || odd(out)) return DLM_ERR_ALIGN;
    return done(launch_head_merge(dtype, head_of(s), head_rows_of(r), nsplit, part_o, part_ml, out, ldo, hs(stream)));
}

int dlm_short_conv(int dtype, const dlm_short_conv_args *c, void *act, void *stream) {
    const int e = check_conv(dtype, c, act);
    return e ? e : done(launch_short_conv(dtype, conv_of(c), c->proj, c->history, act, hs(stream)));
}

int dlm_head_state_begin(int dtype, const dlm_head_shape *s, const dlm_head_rows *r, void *q, const dlm_recurrence_args *a, float *o, void *stream) {
    int c = check_head(dtype, s, r);
    if (!c) c = check_recurrence(dtype, a);
    if (c) return c;
    if (!q || !o) return DLM_ERR_NULL;
    if (r->M != 1 || a->M != 1 || a->z) return DLM_ERR_SHAPE;
    if (odd(q) || odd(o)) return DLM_ERR_ALIGN;
    return done(launch_head_state_begin(dtype, head_of(s), head_rows_of(r), q, linear_of(a), o, hs(stream)));
}

int dlm_head_state_end(int dtype, const dlm_head_shape *s, const dlm_head_rows *r, int nsplit, const float *part_o, const float *part_ml, void *out,
                       const float *o, const float *w, const void *gate, int cols, int true_cols, float eps, void *norm_out, void *stream) {
    const int c = check_head(dtype, s, r);
    if (c) return c;
    if (!part_o || !part_ml || !out || !o || !w || !gate || !norm_out) return DLM_ERR_NULL;
    if (r->M != 1 || nsplit <= 0 || nsplit > 256 || !decode_block_keys(dtype, head_view(head_of(s))) || cols <= 0 || cols % 4 || true_cols <= 0 ||
        true_cols > cols || !(eps >= 0.f))
        return DLM_ERR_SHAPE;
    if (odd(part_o) || odd(out) || odd(o) || odd(w)) return DLM_ERR_ALIGN;
    return done(launch_head_state_end(dtype, head_of(s), head_rows_of(r), nsplit, part_o, part_ml, out, GatedNorm{o, 1, cols, true_cols, w, eps, cols, cols}, gate,
                                      norm_out, hs(stream)));
}

int dlm_conv_products(int dtype, const dlm_short_conv_args *c, void *act, const dlm_short_product *a, const dlm_short_product *b, void *stream) {
    const int e = check_conv(dtype, c, act);
    if (e) return e;
    if (c->M != 1) return DLM_ERR_SHAPE;
    for (const dlm_short_product *p : {a, b}) {
        if (!p || !p->w || !p->x || !p->out) return DLM_ERR_NULL;
        if (p->K <= 0 || p->K % 64 || p->N <= 0 || p->N % 16) return DLM_ERR_SHAPE;
        if (odd(p->w) || odd(p->x)) return DLM_ERR_ALIGN;
    }
    return done(launch_conv_products(dtype, conv_of(c), c->proj, c->history, act, ShortProduct{a->w, a->x, a->out, a->K, a->N},
                                     ShortProduct{b->w, b->x, b->out, b->K, b->N}, hs(stream)));
}

int dlm_recurrence_steps(int dtype, const dlm_recurrence_args *a, float *o, void *stream) {
    const int c = check_recurrence(dtype, a);
    if (c) return c;
    if (!o) return DLM_ERR_NULL;
    return done(launch_recurrence_steps(dtype, linear_of(a), o, hs(stream)));
}

size_t dlm_recurrence_chunk_bytes(const dlm_recurrence_args *a) {
    return a && a->heads > 0 && a->dim > 0 && a->vdim > 0 && a->M > 0 && linear_chunks_supported(linear_of(a)) ? linear_chunk_bytes(linear_of(a)) : 0;
}

int dlm_recurrence_chunks(int dtype, const dlm_recurrence_args *a, void *work, float *o, void *stream) {
    const int c = check_recurrence(dtype, a);
    if (c) return c;
    if (!work || !o) return DLM_ERR_NULL;
    if (!linear_chunks_supported(linear_of(a))) return DLM_ERR_SHAPE;
    if (odd(work) || odd(o)) return DLM_ERR_ALIGN;
    return done(launch_linear_chunks(dtype, linear_of(a), work, o, hs(stream)));
}

int dlm_gated_norm(int dtype, const float *o, const float *w, const void *gate, int64_t ld_gate, void *out, int64_t ld_out, int M, int groups, int cols,
                   int true_cols, float eps, void *stream) {
    if (!o || !w || !gate || !out) return DLM_ERR_NULL;
    if (bad_type(dtype) || M <= 0 || M > 65535 || groups <= 0 || cols <= 0 || cols % 4 || true_cols <= 0 || true_cols > cols || !(eps >= 0.f) || ld_gate % 4 || ld_out % 4 ||
        ld_out < (int64_t)groups * cols)
        return DLM_ERR_SHAPE;
    if (odd(o) || odd(w)) return DLM_ERR_ALIGN;
    return done(launch_gated_norm(dtype, GatedNorm{o, groups, cols, true_cols, w, eps, (long)ld_gate, (long)ld_out}, gate, out, M, hs(stream)));
}

int dlm_latent_decode_supported(int dtype, const dlm_latent_shape *s) { return s && !bad_type(dtype) && latent_decode_supported(dtype, shape_of(s)); }
int dlm_latent_prefill_supported(int dtype, const dlm_latent_shape *s) { return s && !bad_type(dtype) && latent_prefill_supported(dtype, shape_of(s)); }

int dlm_latent_prepare(int dtype, const dlm_latent_shape *s, const dlm_latent_rows *r, void *stream) {
    const int c = check_latent(dtype, s, r);
    return c ? c : done(launch_latent_prepare(dtype, shape_of(s), rows_of(r), hs(stream)));
}

int dlm_latent_prefill(int dtype, const dlm_latent_shape *s, const dlm_latent_rows *r, const void *kv, int64_t ldkv, const float *sink, void *out,
                       int64_t ldo, void *stream) {
    const int c = check_latent(dtype, s, r);
    if (c) return c;
    if (!kv || !sink || !out) return DLM_ERR_NULL;
    if (r->pos_dev || !latent_prefill_supported(dtype, shape_of(s)) || ldkv % 8 || ldkv < (int64_t)s->heads * (s->dim + s->vdim) || ldo % 8 ||
        ldo < (int64_t)s->heads * s->vdim)
        return DLM_ERR_SHAPE;
    if (odd(kv) || odd(out)) return DLM_ERR_ALIGN;
    return done(launch_latent_prefill(dtype, shape_of(s), rows_of(r), kv, ldkv, sink, out, ldo, hs(stream)));
}

int dlm_latent_absorb(int dtype, const dlm_latent_shape *s, const dlm_latent_rows *r, const void *w_uk, void *qa, void *stream) {
    const int c = check_latent(dtype, s, r);
    if (c) return c;
    if (!w_uk || !qa) return DLM_ERR_NULL;
    if (!latent_decode_supported(dtype, shape_of(s))) return DLM_ERR_SHAPE;
    if (odd(w_uk) || odd(qa)) return DLM_ERR_ALIGN;
    return done(launch_latent_absorb(dtype, shape_of(s), rows_of(r), w_uk, qa, hs(stream)));
}

int dlm_latent_decode(int dtype, const dlm_latent_shape *s, const dlm_latent_rows *r, const void *qa, int nsplit, float *part_o, float *part_ml,
                      void *stream) {
    const int c = check_latent(dtype, s, r);
    if (c) return c;
    if (!qa || !part_o || !part_ml) return DLM_ERR_NULL;
    if (nsplit <= 0 || nsplit > 256 || !latent_decode_supported(dtype, shape_of(s))) return DLM_ERR_SHAPE;
    if (odd(qa) || odd(part_o)) return DLM_ERR_ALIGN;
    return done(launch_latent_decode(dtype, shape_of(s), rows_of(r), qa, nsplit, part_o, part_ml, hs(stream)));
}

int dlm_latent_combine(int dtype, const dlm_latent_shape *s, const dlm_latent_rows *r, int nsplit, const float *part_o, const float *part_ml,
                       const float *sink, const void *w_uv, void *out, int64_t ldo, void *stream) {
    const int c = check_latent(dtype, s, r);
    if (c) return c;
    if (!part_o || !part_ml || !sink || !w_uv || !out) return DLM_ERR_NULL;
    if (nsplit <= 0 || nsplit > 256 || !latent_decode_supported(dtype, shape_of(s)) || ldo < (int64_t)s->heads * s->vdim) return DLM_ERR_SHAPE;
    if (odd(part_o) || odd(w_uv)) return DLM_ERR_ALIGN;
    return done(launch_latent_combine(dtype, shape_of(s), rows_of(r), nsplit, part_o, part_ml, sink, w_uv, out, ldo, hs(stream)));
}

}  // extern "C"
