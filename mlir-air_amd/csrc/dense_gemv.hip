// One-token products with dense weights for gfx950: y[N] = W[N, K] x[K], W row-major in the element type.
//
// HBM-bound: every byte of W is read once.  A wavefront owns R consecutive rows at a time and reads each as coalesced
// 1 KiB pieces (8 consecutive k per lane), R x U of them in flight; x lies in LDS in the element type.  The row sums are
// fp32, added over the 64 lanes by a butterfly.  The workgroups walk the rows with a stride (at most kMaxBlocks of them),
// so that what a workgroup does to get x is done once per workgroup and not once per row group.
//
// The intake computes x where another kernel would otherwise be launched for it: the embedding row, or the residual
// stream with the normed output of the previous sublayer added (every workgroup redoes this small sum from L2; one of
// them stores it), or the final norm of that, or the norm of the stream with the previous sublayer's output added.  The first
// weights are requested before it.  The row sums can be combined in pairs: activation of a gate row times an up row.
#include "dense.h"
#include "dense_kernels.h"

namespace w4a16 {

namespace {

constexpr int kGemvWaves = 4, kGemvThreads = 64 * kGemvWaves;
constexpr int kMaxBlocks = 1024;
constexpr int kPiece = 512;   // elements of a row that a wave reads at once

template <class T>
struct GemvParams {
    const T *w;
    T *out;
    float *out_f32;
    unsigned long long *keys;
    int n_valid, K, N, groups;
    const T *x;
    const float *res, *y, *norm_w, *final_w;
    float eps;
    int width;
    float *res_out;
    T *h_out;
    const T *embed;
    const int32_t *token;
    float scale;
    RowOutput ro;
};

// sum over the workgroup, for every thread
__device__ __forceinline__ float block_sum(float v, float *red) {
    v = wave_reduce<false>(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = red[0];
#pragma unroll
    for (int i = 1; i < kGemvWaves; ++i) s += red[i];
    return s;
}

// x into LDS (K elements, zeros up to the next piece)
template <class T, int MODE>
__device__ __forceinline__ void take_in(const GemvParams<T> &p, T *xs, float *red) {
    const int tid = threadIdx.x;
    const int kl = (p.K + kPiece - 1) / kPiece * kPiece;
    for (int i = p.K + 8 * tid; i < kl; i += 8 * kGemvThreads) store8(xs + i, zero8<T>());
    if constexpr (MODE == kIntakePlain) {
        for (int i = 8 * tid; i < p.K; i += 8 * kGemvThreads) store8(xs + i, load8(p.x + i));
    } else if constexpr (MODE == kIntakeEmbed) {
        const T *row = p.embed + (size_t)p.token[0] * p.K;
        for (int i = 4 * tid; i < p.K; i += 4 * kGemvThreads) {
            float e[4];
            load4(row + i, e);
#pragma unroll
            for (int j = 0; j < 4; ++j) e[j] *= p.scale;
            store4(xs + i, e[0], e[1], e[2], e[3]);
            if (blockIdx.x == 0) {
                store4(p.res_out + i, e[0], e[1], e[2], e[3]);
                if (p.h_out) store4(p.h_out + i, e[0], e[1], e[2], e[3]);
            }
        }
    } else if constexpr (MODE == kIntakeNormed) {
        const T *row = p.embed ? p.embed + (size_t)p.token[0] * p.K : nullptr;
        auto value = [&](int i, float (&v)[4]) {
            if (row) {
                load4(row + i, v);
#pragma unroll
                for (int j = 0; j < 4; ++j) v[j] *= p.scale;
                return;
            }
            load4(p.res + i, v);
            if (p.y) {
                float u[4];
                load4(p.y + i, u);
#pragma unroll
                for (int j = 0; j < 4; ++j) v[j] += u[j];
            }
        };
        float ss = 0.f;
        for (int i = 4 * tid; i < p.K; i += 4 * kGemvThreads) {
            float v[4];
            value(i, v);
#pragma unroll
            for (int j = 0; j < 4; ++j) ss = fmaf(v[j], v[j], ss);
            if (blockIdx.x == 0 && p.res_out) store4(p.res_out + i, v[0], v[1], v[2], v[3]);
        }
        const float rstd = 1.0f / sqrtf(block_sum(ss, red) / (float)p.width + p.eps);
        for (int i = 4 * tid; i < p.K; i += 4 * kGemvThreads) {
            float v[4], w[4];
            value(i, v);
            load4(p.final_w + i, w);
            store4(xs + i, v[0] * rstd * w[0], v[1] * rstd * w[1], v[2] * rstd * w[2], v[3] * rstd * w[3]);
        }
    } else {
        float rstd = 0.f;
        if (p.y) {
            float ss = 0.f;
            for (int i = 4 * tid; i < p.K; i += 4 * kGemvThreads) {
                float v[4];
                load4(p.y + i, v);
#pragma unroll
                for (int j = 0; j < 4; ++j) ss = fmaf(v[j], v[j], ss);
            }
            rstd = 1.0f / sqrtf(block_sum(ss, red) / (float)p.width + p.eps);
        }
        auto value = [&](int i, float (&v)[4]) {
            load4(p.res + i, v);
            if (p.y) {
                float u[4], w[4];
                load4(p.y + i, u);
                load4(p.norm_w + i, w);
#pragma unroll
                for (int j = 0; j < 4; ++j) v[j] = fmaf(u[j] * rstd, w[j], v[j]);
            }
        };
        if constexpr (MODE == kIntakeResidual) {
            for (int i = 4 * tid; i < p.K; i += 4 * kGemvThreads) {
                float v[4];
                value(i, v);
                store4(xs + i, v[0], v[1], v[2], v[3]);
                if (blockIdx.x == 0) {
                    if (p.res_out) store4(p.res_out + i, v[0], v[1], v[2], v[3]);
                    if (p.h_out) store4(p.h_out + i, v[0], v[1], v[2], v[3]);
                }
            }
        } else {
            float ss = 0.f;
            for (int i = 4 * tid; i < p.K; i += 4 * kGemvThreads) {
                float v[4];
                value(i, v);
#pragma unroll
                for (int j = 0; j < 4; ++j) ss = fmaf(v[j], v[j], ss);
            }
            const float r2 = 1.0f / sqrtf(block_sum(ss, red) / (float)p.width + p.eps);
            for (int i = 4 * tid; i < p.K; i += 4 * kGemvThreads) {
                float v[4], w[4];
                value(i, v);
                load4(p.final_w + i, w);
                store4(xs + i, v[0] * r2 * w[0], v[1] * r2 * w[1], v[2] * r2 * w[2], v[3] * r2 * w[3]);
            }
        }
    }
}

// (PAIR: rows 2 o and 2 o + 1 of the walk are the gate and the up row of output o)
template <class T, int R, int U, bool PAIR>
__device__ __forceinline__ void request(Vec8<T> (&w)[R][U], const T *base, int K, int N, int row0, int c0) {
    const int lane = threadIdx.x & 63;
#pragma unroll
    for (int r = 0; r < R; ++r) {
        int row = row0 + r < N ? row0 + r : N - 1;   // past the end: read in range, never stored
        if constexpr (PAIR) row = (row >> 5) * 32 + ((row & 31) >> 1) + 16 * (row & 1);
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int k = (c0 + u) * kPiece + 8 * lane;
            w[r][u] = k < K ? stream8(base + (size_t)row * K + k) : zero8<T>();
        }
    }
}

template <class T, int R, int U, int MODE, bool PAIR>
__global__ void __launch_bounds__(kGemvThreads) dense_gemv_kernel(const GemvParams<T> p) {
    extern __shared__ __attribute__((aligned(16))) char gemv_lds[];
    __shared__ float red[kGemvWaves];
    T *xs = reinterpret_cast<T *>(gemv_lds);
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int stride = gridDim.x * kGemvWaves;
    const int pieces = (p.K + kPiece - 1) / kPiece;
    int g = blockIdx.x * kGemvWaves + wave;
    Vec8<T> w[R][U];
    if (g < p.groups) request<T, R, U, PAIR>(w, p.w, p.K, p.N, g * R, 0);
    take_in<T, MODE>(p, xs, red);
    __syncthreads();
    unsigned long long best = 0;
    for (; g < p.groups; g += stride) {
        float acc[R];
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r] = 0.f;
        for (int c0 = 0; c0 < pieces; c0 += U) {
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int c = c0 + u < pieces ? c0 + u : pieces - 1;   // (weights past the last piece are zeros)
                const Vec8<T> xv = load8(xs + c * kPiece + 8 * lane);
#pragma unroll
                for (int r = 0; r < R; ++r) acc[r] = dot8(w[r][u], xv, acc[r]);
            }
            if (c0 + U < pieces) request<T, R, U, PAIR>(w, p.w, p.K, p.N, g * R, c0 + U);
        }
        if (g + stride < p.groups) request<T, R, U, PAIR>(w, p.w, p.K, p.N, (g + stride) * R, 0);
        float mine = 0.f;
        if constexpr (PAIR) {
#pragma unroll
            for (int r = 0; r < R; r += 2) {
                const float a = wave_reduce<false>(acc[r]), b = wave_reduce<false>(acc[r + 1]);
                mine = lane == r / 2 ? (p.ro.gate == kGateGelu ? gelu_tanh_f32(a) : silu_f32(a)) * b : mine;
            }
            const int o = g * (R / 2) + lane;
            if (lane < R / 2 && 2 * o < p.N) p.out[o] = from_float<T>(mine);
            continue;
        }
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const float s = wave_reduce<false>(acc[r]);
            mine = lane == r ? s : mine;
        }
        const int row = g * R + lane;
        if (lane < R && row < p.N) {
            if (row >= p.ro.silu_begin && row < p.ro.silu_end) mine = silu_f32(mine);
            if (p.out_f32) p.out_f32[row] = mine;
            else p.out[row] = from_float<T>(mine);
            if (p.keys && row < p.n_valid) {
                const unsigned long long key = ((unsigned long long)order_key(mine) << 32) | (0xFFFFFFFFu - (uint32_t)row);
                best = key > best ? key : best;
            }
        }
    }
    if (p.keys) {
        best = wave_max_u64(best);
        if (lane == 0) p.keys[blockIdx.x * kGemvWaves + wave] = best;
    }
}

__global__ void __launch_bounds__(1024) argmax_keys_kernel(const unsigned long long *keys, int n, int32_t *token, int32_t *position,
                                                           int32_t *history) {
    __shared__ unsigned long long part[16];
    unsigned long long best = 0;
    for (int i = threadIdx.x; i < n; i += 1024) best = keys[i] > best ? keys[i] : best;
    best = wave_max_u64(best);
    if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = best;
    __syncthreads();
    if (threadIdx.x == 0) {
#pragma unroll
        for (int i = 1; i < 16; ++i) best = part[i] > best ? part[i] : best;
        const int32_t id = (int32_t)(0xFFFFFFFFu - (uint32_t)(best & 0xFFFFFFFFull));
        if (token) token[0] = id;
        if (position) {
            const int32_t next = position[0] + 1;   // the position of the chosen token
            position[0] = next;
            if (history) history[next] = id;
        }
    }
}

template <class T, int R, int U>
hipError_t launch_mode(const GemvParams<T> &p, int mode, int grid, size_t lds, hipStream_t stream) {
    auto run = [&](auto kernel) {
        if (lds > 48 * 1024) {
            const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
            if (e != hipSuccess) return e;
        }
        hipLaunchKernelGGL(kernel, dim3(grid), dim3(kGemvThreads), lds, stream, p);
        return hipGetLastError();
    };
    if (p.ro.gate) {
        if constexpr (R >= 2)
            return mode == kIntakeNormed ? run(&dense_gemv_kernel<T, R, U, kIntakeNormed, true>) : run(&dense_gemv_kernel<T, R, U, kIntakePlain, true>);
        return hipErrorInvalidValue;
    }
    switch (mode) {
        case kIntakePlain: return run(&dense_gemv_kernel<T, R, U, kIntakePlain, false>);
        case kIntakeResidual: return run(&dense_gemv_kernel<T, R, U, kIntakeResidual, false>);
        case kIntakeEmbed: return run(&dense_gemv_kernel<T, R, U, kIntakeEmbed, false>);
        case kIntakeNormed: return run(&dense_gemv_kernel<T, R, U, kIntakeNormed, false>);
        default: return run(&dense_gemv_kernel<T, R, U, kIntakeFinal, false>);
    }
}

int rows_per_wave(int K, int N) { return K > 2048 || N < 512 ? 1 : K > 1024 ? 2 : 4; }

template <class T>
hipError_t launch_typed(const void *w, const RowIntake &in, void *out, float *out_f32, unsigned long long *keys, int n_valid, int K, int N,
                        const RowOutput &ro, hipStream_t stream) {
    GemvParams<T> p;
    p.ro = ro;
    p.w = static_cast<const T *>(w);
    p.out = static_cast<T *>(out);
    p.out_f32 = out_f32;
    p.keys = keys;
    p.n_valid = n_valid;
    p.K = K;
    p.N = N;
    p.x = static_cast<const T *>(in.x);
    p.res = in.res;
    p.y = in.y;
    p.norm_w = in.norm_w;
    p.final_w = in.final_w;
    p.eps = in.eps;
    p.width = in.width;
    p.res_out = in.res_out;
    p.h_out = static_cast<T *>(in.h_out);
    p.embed = static_cast<const T *>(in.embed);
    p.token = in.token;
    p.scale = in.scale;
    const int R = ro.gate && K > 1024 ? 2 : ro.gate ? 4 : rows_per_wave(K, N);
    p.groups = (N + R - 1) / R;
    const int need = (p.groups + kGemvWaves - 1) / kGemvWaves, grid = need < kMaxBlocks ? need : kMaxBlocks;
    const size_t lds = (size_t)((K + kPiece - 1) / kPiece) * kPiece * sizeof(T);
    switch (R) {
        case 1: return launch_mode<T, 1, 8>(p, in.mode, grid, lds, stream);
        case 2: return launch_mode<T, 2, 4>(p, in.mode, grid, lds, stream);
        default: return launch_mode<T, 4, 2>(p, in.mode, grid, lds, stream);
    }
}

}  // namespace

int dense_gemv_blocks(int K, int N) {
    const int R = rows_per_wave(K, N), per = R * kGemvWaves;
    const int need = (N + per - 1) / per;
    return need < kMaxBlocks ? need : kMaxBlocks;
}

hipError_t launch_dense_gemv(int dtype, const void *w, const RowIntake &in, void *out, float *out_f32, unsigned long long *keys, int n_valid,
                             int K, int N, hipStream_t stream, const RowOutput &ro) {
    return dtype == kF32 ? launch_typed<float>(w, in, out, out_f32, keys, n_valid, K, N, ro, stream)
                         : launch_typed<bf16>(w, in, out, out_f32, keys, n_valid, K, N, ro, stream);
}

hipError_t launch_argmax_keys(const unsigned long long *keys, int n, int32_t *token, int32_t *position, int32_t *history, hipStream_t stream) {
    hipLaunchKernelGGL(argmax_keys_kernel, dim3(1), dim3(1024), 0, stream, keys, n, token, position, history);
    return hipGetLastError();
}

}  // namespace w4a16
