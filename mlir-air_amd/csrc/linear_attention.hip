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
#include "mixer_steps.h"

namespace w4a16 {

namespace {

// blockIdx.y: kConvTokens tokens
template <class T>
__global__ void __launch_bounds__(kStepThreads) short_conv_kernel(const ConvArgs c, const T *proj, T *history, T *act, int lanes) {
    short_conv_step<T>(c, proj, history, act, lanes, blockIdx.x, blockIdx.y * kConvTokens);
}

// the last rows of a portion into the history (a launch of its own: short_conv reads the rows that this overwrites)
template <class T>
__global__ void __launch_bounds__(kStepThreads) conv_history_kernel(const ConvArgs c, const T *proj, T *history) {
    const int C = 2 * c.k_heads * c.dim + c.heads * c.vdim, ch = 4 * (blockIdx.x * kStepThreads + threadIdx.x), m = c.M - 1 - (int)blockIdx.y;
    if (ch >= C || m < 0) return;
    float x[4];
    load4(proj + (size_t)m * c.ld + ch, x);
    store4(history + (size_t)((c.pos + m) % c.taps) * C + ch, x[0], x[1], x[2], x[3]);
}

// blockIdx.x = 16 value columns, blockIdx.y = head
template <class T, int ND, bool DELTA>
__global__ void __launch_bounds__(kStepThreads) recurrence_steps_kernel(const LinearArgs a, float *o) {
    recurrence_step<T, ND, DELTA>(a, o, blockIdx.y, blockIdx.x);
}

// Short groups (a head): by `lanes` lanes each; blockIdx.y = token.
template <class T>
__global__ void __launch_bounds__(kStepThreads) gated_norm_heads_kernel(const GatedNorm g, const T *gate, T *out, int lanes) {
    const int lane = threadIdx.x % lanes, grp = blockIdx.x * (kStepThreads / lanes) + threadIdx.x / lanes;
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
__global__ void __launch_bounds__(kStepThreads) gated_norm_row_kernel(const GatedNorm g, const T *gate, T *out) {
    __shared__ float red[4];
    gated_norm_row_step<T>(g, gate, out, blockIdx.x, red);
}

template <class T>
hipError_t conv(const ConvArgs &c, const void *proj, void *history, void *act, hipStream_t stream) {
    const int lanes = lanes_of(c.dim > c.vdim ? c.dim : c.vdim, 8), per = kStepThreads / lanes, units = 2 * c.k_heads + c.heads;
    const T *x = static_cast<const T *>(proj) + c.off;
    hipLaunchKernelGGL(short_conv_kernel<T>, dim3((units + per - 1) / per, (c.M + kConvTokens - 1) / kConvTokens), dim3(kStepThreads), 0, stream, c, x,
                       static_cast<T *>(history), static_cast<T *>(act), lanes);
    const hipError_t e = hipGetLastError();
    if (e != hipSuccess || c.M == 1) return e;
    const int C = 2 * c.k_heads * c.dim + c.heads * c.vdim, rows = c.M < c.taps ? c.M : c.taps;
    hipLaunchKernelGGL(conv_history_kernel<T>, dim3((C / 4 + kStepThreads - 1) / kStepThreads, rows), dim3(kStepThreads), 0, stream, c, x, static_cast<T *>(history));
    return hipGetLastError();
}

template <class T, bool DELTA>
hipError_t steps(const LinearArgs &a, float *o, hipStream_t stream) {
    const dim3 grid(a.vdim / 16, a.heads);
    auto run = [&](auto kernel) {
        hipLaunchKernelGGL(kernel, grid, dim3(kStepThreads), 0, stream, a, o);
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
    const int lanes = lanes_of(g.cols, 4), per = kStepThreads / lanes;
    const dim3 grid = row ? dim3(M) : dim3((g.groups + per - 1) / per, M);
    auto run = [&](auto tag) {
        using T = decltype(tag);
        if (row) hipLaunchKernelGGL(gated_norm_row_kernel<T>, grid, dim3(kStepThreads), 0, stream, g, static_cast<const T *>(gate), static_cast<T *>(out));
        else hipLaunchKernelGGL(gated_norm_heads_kernel<T>, grid, dim3(kStepThreads), 0, stream, g, static_cast<const T *>(gate), static_cast<T *>(out), lanes);
        return hipGetLastError();
    };
    return dtype == kF32 ? run(float{}) : run(bf16{});
}

}  // namespace w4a16
