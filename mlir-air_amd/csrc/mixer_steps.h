// The steps around attention and recurrences as device functions of one workgroup each, so that steps of one token that do not
// wait for each other can share a launch (mixer_steps.hip), besides having launches of their own (head_attention.hip,
// linear_attention.hip).
#pragma once

#include "dense.h"
#include "dense_kernels.h"

namespace w4a16 {

constexpr int kStepThreads = 256;

// lanes that share a vector of n elements, `each` elements per lane at a time
__host__ __device__ inline int lanes_of(int n, int each) {
    int l = 1;
    while (l < 64 && each * l < n) l *= 2;
    return l;
}

// Norm and append of token m: vectors (queries, keys, values) by groups of `lanes` lanes, eight elements per lane at a time.
template <class T>
__device__ __forceinline__ void head_prepare_step(const HeadShape &s, const HeadRows &rows, T *q, int lanes, int block, int m) {
    const int position = (rows.pos_dev ? rows.pos_dev[0] : rows.pos) + m, M = rows.M;
    const T *proj = static_cast<const T *>(rows.proj) + rows.off;
    T *cache = static_cast<T *>(rows.cache);
    const int lane = threadIdx.x % lanes, unit = block * (kStepThreads / lanes) + threadIdx.x / lanes;
    const int H = s.heads, G = s.kv_heads, group = H / G, row_len = s.dim + s.vdim;
    if (unit >= H + 2 * G) return;
    const bool is_q = unit < H, is_v = unit >= H + G;
    const T *src = proj + (size_t)m * rows.ld + (is_v ? (size_t)(H + G) * s.dim + (size_t)(unit - H - G) * s.vdim : (size_t)unit * s.dim);
    const int n = is_v ? s.vdim : s.dim;
    const int g = is_q ? unit / group : is_v ? unit - H - G : unit - H;
    T *row = cache + ((size_t)g * s.ring + position % s.ring) * row_len;
    T *dst = is_q ? q + (((size_t)g * M + m) * group + unit % group) * s.dim : is_v ? row + s.dim : row;
    float rstd = 1.f;
    if (!is_v) {
        float ss = 0.f;
        for (int i = 8 * lane; i < n; i += 8 * lanes) {
            float v[8];
            unpack8(load8(src + i), v);
#pragma unroll
            for (int j = 0; j < 8; ++j) ss = fmaf(v[j], v[j], ss);
        }
        rstd = 1.0f / sqrtf(group_sum(ss, lanes) / (float)s.true_dim + rows.eps);
    }
    const float *w = is_q ? rows.q_norm : rows.k_norm;
    for (int i = 8 * lane; i < n; i += 8 * lanes) {
        const Vec8<T> x = load8(src + i);
        if (is_v) {
            store8(dst + i, x);
            continue;
        }
        float v[8], f[8];
        unpack8(x, v);
        unpack8(load8(w + i), f);
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] *= rstd * f[j];
        store8(dst + i, pack8<T>(v));
    }
}

constexpr int kMergeSplits = 256;

// The splits of query head h and token m merged.  part: kStepThreads entries of LDS, f: kMergeSplits, red: 8.
template <class T>
__device__ __forceinline__ void head_merge_step(const HeadShape &s, int M, const int32_t *pos_dev, int pos, int nsplit, int kb, const float *part_o,
                                                const float *part_ml, T *out, long ldo, int h, int m, float *f, float *red, floatx4 *part) {
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int group = s.heads / s.kv_heads;
    const size_t row = ((size_t)(h / group) * M + m) * group + h % group;
    const int pos0 = pos_dev ? pos_dev[0] : pos, n = pos0 + M - first_block_key(pos0, s.window, kb);
    const int per = keys_per_split(n, nsplit, kb), active = (n + per - 1) / per;
    float ms = kAttnNegBig, ls = 0.f;
    if (tid < active) {
        ms = part_ml[(row * nsplit + tid) * 2];
        ls = part_ml[(row * nsplit + tid) * 2 + 1];
    }
    float top = wave_reduce<true>(ms);
    if (lane == 0) red[wave] = top;
    __syncthreads();
    top = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float fac = tid < active ? exp2f(ms - top) : 0.f;
    const float den = wave_reduce<false>(fac * ls);
    if (lane == 0) red[4 + wave] = den;
    f[tid] = fac;
    __syncthreads();
    const float scale = s.out_scale / (red[4] + red[5] + red[6] + red[7]);
    // a thread adds every `ways`-th split of four columns
    for (int c0 = 0; c0 < s.vdim; c0 += 4 * kStepThreads) {
        const int width = (s.vdim - c0) / 4 < kStepThreads ? (s.vdim - c0) / 4 : kStepThreads;   // four-column pieces of this pass
        const int ways = kStepThreads / width, way = tid / width, col = c0 + 4 * (tid % width);
        floatx4 a = floatx4{0.f, 0.f, 0.f, 0.f};
        if (way < ways)
            for (int i = way; i < active; i += ways) a += *reinterpret_cast<const floatx4 *>(part_o + (row * nsplit + i) * s.vdim + col) * f[i];
        part[tid] = a;
        __syncthreads();
        if (way == 0) {
            for (int w = 1; w < ways; ++w) a += part[tid + w * width];
            a *= scale;
            store4(out + (size_t)m * ldo + (size_t)h * s.vdim + col, a[0], a[1], a[2], a[3]);
        }
        __syncthreads();
    }
}

constexpr int kConvTokens = 4;   // tokens per thread

// Vectors (q and k heads, then v heads) by groups of `lanes` lanes, eight channels per lane at a time; tokens m0 .. m0 + kConvTokens - 1.
// Rows in front of the portion come from the history, a ring of `taps` rows by position.
template <class T>
__device__ __forceinline__ void short_conv_step(const ConvArgs &c, const T *proj, T *history, T *act, int lanes, int block, int m0) {
    const int lane = threadIdx.x % lanes, unit = block * (kStepThreads / lanes) + threadIdx.x / lanes;
    const int units = 2 * c.k_heads + c.heads, C = 2 * c.k_heads * c.dim + c.heads * c.vdim;
    if (unit >= units) return;
    const bool is_v = unit >= 2 * c.k_heads;
    const int c0 = is_v ? 2 * c.k_heads * c.dim + (unit - 2 * c.k_heads) * c.vdim : unit * c.dim, n = is_v ? c.vdim : c.dim;
    const int pos0 = c.pos_dev ? c.pos_dev[0] : c.pos;
    const bool inside = m0 >= c.taps - 1 && m0 + kConvTokens <= c.M;   // every row is one of the portion
    float ss[kConvTokens] = {0.f, 0.f, 0.f, 0.f};
    for (int i = 8 * lane; i < n; i += 8 * lanes) {
        const int ch = c0 + i;
        float acc[kConvTokens][8];
#pragma unroll
        for (int t = 0; t < kConvTokens; ++t)
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[t][e] = 0.f;
        if (inside) {
            for (int j = 0; j < c.taps; ++j) {
                const T *row = proj + (size_t)(m0 + j - (c.taps - 1)) * c.ld + ch;
                float w[8];
                unpack8(load8(c.w + (size_t)j * C + ch), w);
                Vec8<T> v[kConvTokens];
#pragma unroll
                for (int t = 0; t < kConvTokens; ++t) v[t] = load8(row + (size_t)t * c.ld);
#pragma unroll
                for (int t = 0; t < kConvTokens; ++t) {
                    float x[8];
                    unpack8(v[t], x);
#pragma unroll
                    for (int e = 0; e < 8; ++e) acc[t][e] = fmaf(w[e], x[e], acc[t][e]);
                }
            }
        } else {
            for (int j = 0; j < c.taps; ++j) {
                float w[8];
                unpack8(load8(c.w + (size_t)j * C + ch), w);
#pragma unroll
                for (int t = 0; t < kConvTokens; ++t) {
                    const int m = m0 + t, r = m + j - (c.taps - 1);       // row of the portion that meets this tap
                    if (m >= c.M || pos0 + r < 0) continue;
                    float x[8];
                    unpack8(load8(r >= 0 ? proj + (size_t)r * c.ld + ch : history + (size_t)((pos0 + r) % c.taps) * C + ch), x);
#pragma unroll
                    for (int e = 0; e < 8; ++e) acc[t][e] = fmaf(w[e], x[e], acc[t][e]);
                }
            }
        }
#pragma unroll
        for (int t = 0; t < kConvTokens; ++t) {
            if (m0 + t >= c.M) continue;
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[t][e] *= sigmoid_of<T>(acc[t][e]);
            const Vec8<T> out = pack8<T>(acc[t]);
            store8(act + (size_t)(m0 + t) * C + ch, out);
            unpack8(out, acc[t]);   // (the norm is that of what is stored)
#pragma unroll
            for (int e = 0; e < 8; ++e) ss[t] = fmaf(acc[t][e], acc[t][e], ss[t]);
        }
        if (c.M == 1) store8(history + (size_t)(pos0 % c.taps) * C + ch, load8(proj + ch));   // (nobody else reads these channels, nor this slot)
    }
    if (is_v) return;
#pragma unroll
    for (int t = 0; t < kConvTokens; ++t) {
        const float s = group_sum(ss[t], lanes);
        if (lane == 0 && m0 + t < c.M)
            c.factors[(size_t)(m0 + t) * 2 * c.k_heads + unit] = 1.0f / sqrtf(s + c.unit_eps) * (unit < c.k_heads ? c.q_scale : 1.0f);
    }
}

// 16 value columns (`tile`) of head h.  A value column lies in the 16 lanes of a DPP row, lane l holding the channels
// 64 c + 4 l .. + 3.
template <class T, int ND, bool DELTA>
__device__ __forceinline__ void recurrence_step(const LinearArgs &a, float *o, int h, int tile) {
    const T *q = static_cast<const T *>(a.qkv) + a.q_off, *k = static_cast<const T *>(a.qkv) + a.k_off, *v = static_cast<const T *>(a.qkv) + a.v_off;
    const T *beta = static_cast<const T *>(a.beta);
    const int col = tile * 16 + (threadIdx.x >> 4), l4 = 4 * (threadIdx.x & 15);
    const int kh = h / (a.heads / a.k_heads), pos0 = a.pos_dev ? a.pos_dev[0] : a.pos;
    float *st = a.state + ((size_t)h * a.vdim + col) * a.dim + l4;
    floatx4 s[ND];
#pragma unroll
    for (int c = 0; c < ND; ++c) s[c] = pos0 > 0 ? *reinterpret_cast<const floatx4 *>(st + 64 * c) : floatx4{0.f, 0.f, 0.f, 0.f};

    float ea = 0.f, g1 = 1.f;
    floatx4 bias[ND];
    if constexpr (DELTA) {
        ea = -expf(a.a_log[h]) * 1.4426950408889634f;
#pragma unroll
        for (int c = 0; c < ND; ++c) bias[c] = *reinterpret_cast<const floatx4 *>(a.dt_bias + (size_t)h * a.dim + 64 * c + l4);
    } else {
        g1 = __builtin_amdgcn_exp2f(a.log2_decay[h]);
    }
    struct Row {
        float q[ND][4], k[ND][4], v, qf, kf, beta;
        floatx4 z[ND];
    };
    auto fetch = [&](int m, Row &r) {
        const T *qr = q + (size_t)m * a.ld + (size_t)kh * a.dim + l4, *kr = k + (size_t)m * a.ld + (size_t)kh * a.dim + l4;
#pragma unroll
        for (int c = 0; c < ND; ++c) {
            load4(qr + 64 * c, r.q[c]);
            load4(kr + 64 * c, r.k[c]);
            if constexpr (DELTA) r.z[c] = *reinterpret_cast<const floatx4 *>(a.z + (size_t)m * a.heads * a.dim + (size_t)h * a.dim + 64 * c + l4);
        }
        r.v = to_float(v[(size_t)m * a.ld + (size_t)h * a.vdim + col]);
        if constexpr (DELTA) {
            r.qf = a.factors[(size_t)m * 2 * a.k_heads + kh];
            r.kf = a.factors[(size_t)m * 2 * a.k_heads + a.k_heads + kh];
            r.beta = to_float(beta[(size_t)m * a.ld_beta + h]);
        }
    };
    Row cur;
    fetch(0, cur);
    for (int m = 0; m < a.M; ++m) {
        Row next;
        fetch(m + 1 < a.M ? m + 1 : m, next);
        float u = cur.v;
        if constexpr (DELTA) {
            float p = 0.f;
#pragma unroll
            for (int c = 0; c < ND; ++c)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    s[c][e] *= __builtin_amdgcn_exp2f(ea * softplus_f32(cur.z[c][e] + bias[c][e]));
                    cur.k[c][e] *= cur.kf;
                    cur.q[c][e] *= cur.qf;
                    p = fmaf(s[c][e], cur.k[c][e], p);
                }
            u = sigmoid_f32(cur.beta) * (u - row_sum16(p));
        }
        float r = 0.f;
#pragma unroll
        for (int c = 0; c < ND; ++c)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                s[c][e] = fmaf(cur.k[c][e], u, DELTA ? s[c][e] : s[c][e] * g1);
                r = fmaf(s[c][e], cur.q[c][e], r);
            }
        r = row_sum16(r);
        if (l4 == 0) o[(size_t)m * a.heads * a.vdim + (size_t)h * a.vdim + col] = r;
        cur = next;
    }
#pragma unroll
    for (int c = 0; c < ND; ++c) *reinterpret_cast<floatx4 *>(st + 64 * c) = s[c];
}

// One long group, token m.  red: 4 floats of LDS.
template <class T>
__device__ __forceinline__ void gated_norm_row_step(const GatedNorm &g, const T *gate, T *out, size_t m, float *red) {
    const float *o = g.o + m * g.cols;
    float ss = 0.f;
    for (int i = 4 * threadIdx.x; i < g.cols; i += 4 * kStepThreads) {
        const floatx4 v = *reinterpret_cast<const floatx4 *>(o + i);
#pragma unroll
        for (int j = 0; j < 4; ++j) ss = fmaf(v[j], v[j], ss);
    }
    ss = wave_reduce<false>(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    const float rstd = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)g.true_cols + g.eps);
    for (int i = 4 * threadIdx.x; i < g.cols; i += 4 * kStepThreads) {
        const floatx4 v = *reinterpret_cast<const floatx4 *>(o + i), w = *reinterpret_cast<const floatx4 *>(g.w + i);
        float z[4];
        load4(gate + m * g.ld_gate + i, z);
#pragma unroll
        for (int j = 0; j < 4; ++j) z[j] = v[j] * rstd * w[j] * sigmoid_of<T>(z[j]);
        store4(out + m * g.ld_out + i, z[0], z[1], z[2], z[3]);
    }
}

// out[row] = w[row] x for the rows `row0` .. of this workgroup (kRowsAtOnce per group of `lanes` lanes); x and the rows of w have K elements.
constexpr int kRowsAtOnce = 4;
template <class T, class O>
struct ShortRows {
    const T *w, *x;
    O *out;
    int K, N, lanes, blocks;
};
template <class T, class O>
__device__ __forceinline__ void short_rows_step(const T *w, const T *x, int K, int N, O *out, int lanes, int block) {
    const int lane = threadIdx.x % lanes, row0 = (block * (kStepThreads / lanes) + threadIdx.x / lanes) * kRowsAtOnce;
    if (row0 >= N) return;
    float acc[kRowsAtOnce] = {0.f, 0.f, 0.f, 0.f};
    for (int i = 8 * lane; i < K; i += 8 * lanes) {
        Vec8<T> v[kRowsAtOnce];
#pragma unroll
        for (int r = 0; r < kRowsAtOnce; ++r) v[r] = load8(w + (size_t)(row0 + r) * K + i);   // (N is a multiple of kRowsAtOnce)
        const Vec8<T> xv = load8(x + i);
#pragma unroll
        for (int r = 0; r < kRowsAtOnce; ++r) acc[r] = dot8(v[r], xv, acc[r]);
    }
#pragma unroll
    for (int r = 0; r < kRowsAtOnce; ++r) {
        const float s = group_sum(acc[r], lanes);
        if (lane == 0) out[row0 + r] = from_float<O>(s);
    }
}

}  // namespace w4a16
