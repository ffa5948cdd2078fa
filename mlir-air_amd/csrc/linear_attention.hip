// Linear recurrences over a matrix state per head for gfx950, token by token:
//
//   S <- g * S (one factor per head, or one per key channel);  u = v, or u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
//   short_conv        causal convolution over time per channel, silu, and the factors that make queries and keys unit vectors
//   recurrence_steps  the recurrence of one token or a short portion: HBM-bound on the state, which is read and written once
//   gated_norm        RMS norm of the read-outs (per head or over all heads) times a sigmoid gate
//
// The state is fp32 and stored [head][value column][key channel].  A sequence's first token does not read it.  Long portions
// go through linear_chunks.hip.
#include "dense.h"
#include "dense_kernels.h"

namespace w4a16 {

namespace {

constexpr int kThreads = 256;

// lanes that share a vector of n elements, `each` elements per lane at a time
int lanes_of(int n, int each) {
    int l = 1;
    while (l < 64 && each * l < n) l *= 2;
    return l;
}

constexpr int kConvTokens = 4;   // tokens per thread

// Vectors (q and k heads, then v heads) by groups of `lanes` lanes, eight channels per lane at a time; blockIdx.y: kConvTokens tokens.
// Rows in front of the portion come from the history, a ring of `taps` rows by position.
template <class T>
__global__ void __launch_bounds__(kThreads) short_conv_kernel(const ConvArgs c, const T *proj, T *history, T *act, int lanes) {
    const int lane = threadIdx.x % lanes, unit = blockIdx.x * (kThreads / lanes) + threadIdx.x / lanes;
    const int units = 2 * c.k_heads + c.heads, C = 2 * c.k_heads * c.dim + c.heads * c.vdim;
    if (unit >= units) return;
    const bool is_v = unit >= 2 * c.k_heads;
    const int c0 = is_v ? 2 * c.k_heads * c.dim + (unit - 2 * c.k_heads) * c.vdim : unit * c.dim, n = is_v ? c.vdim : c.dim;
    const int pos0 = c.pos_dev ? c.pos_dev[0] : c.pos, m0 = blockIdx.y * kConvTokens;
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

// the last rows of a portion into the history (a launch of its own: short_conv reads the rows that this overwrites)
template <class T>
__global__ void __launch_bounds__(kThreads) conv_history_kernel(const ConvArgs c, const T *proj, T *history) {
    const int C = 2 * c.k_heads * c.dim + c.heads * c.vdim, ch = 4 * (blockIdx.x * kThreads + threadIdx.x), m = c.M - 1 - (int)blockIdx.y;
    if (ch >= C || m < 0) return;
    float x[4];
    load4(proj + (size_t)m * c.ld + ch, x);
    store4(history + (size_t)((c.pos + m) % c.taps) * C + ch, x[0], x[1], x[2], x[3]);
}

// One workgroup: 16 value columns of a head.  A value column lies in the 16 lanes of a DPP row, lane l holding the channels
// 64 c + 4 l .. + 3.
template <class T, int ND, bool DELTA>
__global__ void __launch_bounds__(kThreads) recurrence_steps_kernel(const LinearArgs a, const T *q, const T *k, const T *v, const T *beta, float *o) {
    const int h = blockIdx.y, col = blockIdx.x * 16 + (threadIdx.x >> 4), l4 = 4 * (threadIdx.x & 15);
    const int kh = h / (a.heads / a.k_heads), pos0 = a.pos_dev ? a.pos_dev[0] : a.pos;
    float *st = a.state + ((size_t)h * a.vdim + col) * a.dim + l4;
    floatx4 s[ND];
#pragma unroll
    for (int c = 0; c < ND; ++c) s[c] = pos0 > 0 ? *reinterpret_cast<const floatx4 *>(st + 64 * c) : floatx4{0.f, 0.f, 0.f, 0.f};

    float ea = 0.f, g1 = 1.f;
    floatx4 bias[ND];
    if constexpr (DELTA) {
        ea = expf(a.a_log[h]);
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
                    s[c][e] *= expf(-ea * softplus_f32(cur.z[c][e] + bias[c][e]));
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

// Short groups (a head): by `lanes` lanes each; blockIdx.y = token.
template <class T>
__global__ void __launch_bounds__(kThreads) gated_norm_heads_kernel(const GatedNorm g, const T *gate, T *out, int lanes) {
    const int lane = threadIdx.x % lanes, grp = blockIdx.x * (kThreads / lanes) + threadIdx.x / lanes;
    if (grp >= g.groups) return;
    const size_t m = blockIdx.y;
    const float *o = g.o + (m * g.groups + grp) * g.cols;
    float ss = 0.f;
    for (int i = 4 * lane; i < g.cols; i += 4 * lanes) {
        const floatx4 v = *reinterpret_cast<const floatx4 *>(o + i);
#pragma unroll
        for (int j = 0; j < 4; ++j) ss = fmaf(v[j], v[j], ss);
    }
    const float rstd = 1.0f / sqrtf(group_sum(ss, lanes) / (float)g.true_cols + g.eps);
    for (int i = 4 * lane; i < g.cols; i += 4 * lanes) {
        const floatx4 v = *reinterpret_cast<const floatx4 *>(o + i), w = *reinterpret_cast<const floatx4 *>(g.w + i);
        float z[4];
        load4(gate + m * g.ld_gate + (size_t)grp * g.cols + i, z);
#pragma unroll
        for (int j = 0; j < 4; ++j) z[j] = v[j] * rstd * w[j] * sigmoid_of<T>(z[j]);
        store4(out + m * g.ld_out + (size_t)grp * g.cols + i, z[0], z[1], z[2], z[3]);
    }
}

// One long group: a workgroup per token.
template <class T>
__global__ void __launch_bounds__(kThreads) gated_norm_row_kernel(const GatedNorm g, const T *gate, T *out) {
    __shared__ float red[4];
    const size_t m = blockIdx.x;
    const float *o = g.o + m * g.cols;
    float ss = 0.f;
    for (int i = 4 * threadIdx.x; i < g.cols; i += 4 * kThreads) {
        const floatx4 v = *reinterpret_cast<const floatx4 *>(o + i);
#pragma unroll
        for (int j = 0; j < 4; ++j) ss = fmaf(v[j], v[j], ss);
    }
    ss = wave_reduce<false>(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    const float rstd = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)g.true_cols + g.eps);
    for (int i = 4 * threadIdx.x; i < g.cols; i += 4 * kThreads) {
        const floatx4 v = *reinterpret_cast<const floatx4 *>(o + i), w = *reinterpret_cast<const floatx4 *>(g.w + i);
        float z[4];
        load4(gate + m * g.ld_gate + i, z);
#pragma unroll
        for (int j = 0; j < 4; ++j) z[j] = v[j] * rstd * w[j] * sigmoid_of<T>(z[j]);
        store4(out + m * g.ld_out + i, z[0], z[1], z[2], z[3]);
    }
}

template <class T>
hipError_t conv(const ConvArgs &c, const void *proj, void *history, void *act, hipStream_t stream) {
    const int lanes = lanes_of(c.dim > c.vdim ? c.dim : c.vdim, 8), per = kThreads / lanes, units = 2 * c.k_heads + c.heads;
    const T *x = static_cast<const T *>(proj) + c.off;
    hipLaunchKernelGGL(short_conv_kernel<T>, dim3((units + per - 1) / per, (c.M + kConvTokens - 1) / kConvTokens), dim3(kThreads), 0, stream, c, x,
                       static_cast<T *>(history), static_cast<T *>(act), lanes);
    const hipError_t e = hipGetLastError();
    if (e != hipSuccess || c.M == 1) return e;
    const int C = 2 * c.k_heads * c.dim + c.heads * c.vdim, rows = c.M < c.taps ? c.M : c.taps;
    hipLaunchKernelGGL(conv_history_kernel<T>, dim3((C / 4 + kThreads - 1) / kThreads, rows), dim3(kThreads), 0, stream, c, x, static_cast<T *>(history));
    return hipGetLastError();
}

template <class T, bool DELTA>
hipError_t steps(const LinearArgs &a, float *o, hipStream_t stream) {
    const dim3 grid(a.vdim / 16, a.heads);
    const T *q = static_cast<const T *>(a.qkv) + a.q_off, *k = static_cast<const T *>(a.qkv) + a.k_off, *v = static_cast<const T *>(a.qkv) + a.v_off;
    auto run = [&](auto kernel) {
        hipLaunchKernelGGL(kernel, grid, dim3(kThreads), 0, stream, a, q, k, v, static_cast<const T *>(a.beta), o);
        return hipGetLastError();
    };
    switch (a.dim / 64) {
        case 1: return run(&recurrence_steps_kernel<T, 1, DELTA>);
        case 2: return run(&recurrence_steps_kernel<T, 2, DELTA>);
        case 3: return run(&recurrence_steps_kernel<T, 3, DELTA>);
        case 4: return run(&recurrence_steps_kernel<T, 4, DELTA>);
        case 5: return run(&recurrence_steps_kernel<T, 5, DELTA>);
        case 6: return run(&recurrence_steps_kernel<T, 6, DELTA>);
        case 7: return run(&recurrence_steps_kernel<T, 7, DELTA>);
        case 8: return run(&recurrence_steps_kernel<T, 8, DELTA>);
        default: return hipErrorInvalidValue;
    }
}

}  // namespace

hipError_t launch_short_conv(int dtype, const ConvArgs &c, const void *proj, void *history, void *act, hipStream_t stream) {
    return dtype == kF32 ? conv<float>(c, proj, history, act, stream) : conv<bf16>(c, proj, history, act, stream);
}

hipError_t launch_recurrence_steps(int dtype, const LinearArgs &a, float *o, hipStream_t stream) {
    if (dtype == kF32) return a.z ? steps<float, true>(a, o, stream) : steps<float, false>(a, o, stream);
    return a.z ? steps<bf16, true>(a, o, stream) : steps<bf16, false>(a, o, stream);
}

hipError_t launch_gated_norm(int dtype, const GatedNorm &g, const void *gate, void *out, int M, hipStream_t stream) {
    const bool row = g.groups == 1 && g.cols > 256;
    const int lanes = lanes_of(g.cols, 4), per = kThreads / lanes;
    const dim3 grid = row ? dim3(M) : dim3((g.groups + per - 1) / per, M);
    auto run = [&](auto tag) {
        using T = decltype(tag);
        if (row) hipLaunchKernelGGL(gated_norm_row_kernel<T>, grid, dim3(kThreads), 0, stream, g, static_cast<const T *>(gate), static_cast<T *>(out));
        else hipLaunchKernelGGL(gated_norm_heads_kernel<T>, grid, dim3(kThreads), 0, stream, g, static_cast<const T *>(gate), static_cast<T *>(out), lanes);
        return hipGetLastError();
    };
    return dtype == kF32 ? run(float{}) : run(bf16{});
}

}  // namespace w4a16
