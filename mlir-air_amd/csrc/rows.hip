// Row-wise steps around the products over many rows: the embedding, the residual sum with the norm of a sublayer's output
// (for experts: with their weighted sum), the norm in front of the head.  The residual is fp32 throughout; one workgroup
// per row.
#include "dense.h"
#include "dense_kernels.h"

namespace w4a16 {

namespace {

constexpr int kRowThreads = 256;

__device__ __forceinline__ float row_total(float v, float *red) {
    v = wave_reduce<false>(v);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return red[0] + red[1] + red[2] + red[3];
}

template <class T>
__global__ void __launch_bounds__(kRowThreads) embed_rows_kernel(const int32_t *tokens, const T *embed, float scale, float *res, T *h, int width) {
    const size_t m = blockIdx.x;
    const T *row = embed + (size_t)tokens[m] * width;
    for (int i = 4 * threadIdx.x; i < width; i += 4 * kRowThreads) {
        float e[4];
        load4(row + i, e);
#pragma unroll
        for (int j = 0; j < 4; ++j) e[j] *= scale;
        store4(res + m * width + i, e[0], e[1], e[2], e[3]);
        store4(h + m * width + i, e[0], e[1], e[2], e[3]);
    }
}

// Y: type of y; top > 0: y holds `top` rows per token, summed with the router's weights (kept in LDS between the passes)
template <class T, class Y>
__global__ void __launch_bounds__(kRowThreads) residual_norm_kernel(float *res, const Y *y, const float *weights, int top, const float *norm_w, float eps,
                                                                    int true_width, T *h, int width) {
    extern __shared__ float sum_lds[];
    __shared__ float red[4];
    const size_t m = blockIdx.x;
    float ss = 0.f;
    for (int i = 4 * threadIdx.x; i < width; i += 4 * kRowThreads) {
        float v[4];
        if (top > 0) {
#pragma unroll
            for (int j = 0; j < 4; ++j) v[j] = 0.f;
            for (int s = 0; s < top; ++s) {
                float u[4];
                load4(y + (m * top + s) * width + i, u);
                const float wt = weights[m * top + s];
#pragma unroll
                for (int j = 0; j < 4; ++j) v[j] = fmaf(wt, u[j], v[j]);
            }
        } else {
            load4(y + m * width + i, v);
        }
        store4(sum_lds + i, v[0], v[1], v[2], v[3]);   // read back by the same thread
#pragma unroll
        for (int j = 0; j < 4; ++j) ss = fmaf(v[j], v[j], ss);
    }
    const float rstd = 1.0f / sqrtf(row_total(ss, red) / (float)true_width + eps);
    for (int i = 4 * threadIdx.x; i < width; i += 4 * kRowThreads) {
        float v[4], w[4], x[4];
        load4(sum_lds + i, v);
        load4(norm_w + i, w);
        load4(res + m * width + i, x);
#pragma unroll
        for (int j = 0; j < 4; ++j) x[j] = fmaf(v[j] * rstd, w[j], x[j]);
        store4(res + m * width + i, x[0], x[1], x[2], x[3]);
        if (h) store4(h + m * width + i, x[0], x[1], x[2], x[3]);
    }
}

template <class T>
__global__ void __launch_bounds__(kRowThreads) norm_rows_kernel(const float *res, const int32_t *rows, const float *norm_w, float eps, int true_width, T *out,
                                                                int width) {
    __shared__ float red[4];
    const float *x = res + (size_t)(rows ? rows[blockIdx.x] : (int)blockIdx.x) * width;
    float ss = 0.f;
    for (int i = 4 * threadIdx.x; i < width; i += 4 * kRowThreads) {
        float v[4];
        load4(x + i, v);
#pragma unroll
        for (int j = 0; j < 4; ++j) ss = fmaf(v[j], v[j], ss);
    }
    const float rstd = 1.0f / sqrtf(row_total(ss, red) / (float)true_width + eps);
    for (int i = 4 * threadIdx.x; i < width; i += 4 * kRowThreads) {
        float v[4], w[4];
        load4(x + i, v);
        load4(norm_w + i, w);
        store4(out + (size_t)blockIdx.x * width + i, v[0] * rstd * w[0], v[1] * rstd * w[1], v[2] * rstd * w[2], v[3] * rstd * w[3]);
    }
}

// the residual brought up to date and its norm: what the sublayers of a model with norms on their inputs read
template <class T>
__global__ void __launch_bounds__(kRowThreads) add_norm_rows_kernel(float *res, const float *y, const int32_t *tokens, const T *embed, float scale,
                                                                    const float *norm_w, float eps, int true_width, T *h, int width) {
    extern __shared__ float sum_lds[];
    __shared__ float red[4];
    const size_t m = blockIdx.x;
    const T *row = tokens ? embed + (size_t)tokens[m] * width : nullptr;
    float ss = 0.f;
    for (int i = 4 * threadIdx.x; i < width; i += 4 * kRowThreads) {
        float v[4];
        if (row) {
            load4(row + i, v);
#pragma unroll
            for (int j = 0; j < 4; ++j) v[j] *= scale;
        } else {
            load4(res + m * width + i, v);
            if (y) {
                float u[4];
                load4(y + m * width + i, u);
#pragma unroll
                for (int j = 0; j < 4; ++j) v[j] += u[j];
            }
        }
        if (row || y) store4(res + m * width + i, v[0], v[1], v[2], v[3]);
        store4(sum_lds + i, v[0], v[1], v[2], v[3]);   // read back by the same thread
#pragma unroll
        for (int j = 0; j < 4; ++j) ss = fmaf(v[j], v[j], ss);
    }
    if (!h) return;
    const float rstd = 1.0f / sqrtf(row_total(ss, red) / (float)true_width + eps);
    for (int i = 4 * threadIdx.x; i < width; i += 4 * kRowThreads) {
        float v[4], w[4];
        load4(sum_lds + i, v);
        load4(norm_w + i, w);
        store4(h + m * width + i, v[0] * rstd * w[0], v[1] * rstd * w[1], v[2] * rstd * w[2], v[3] * rstd * w[3]);
    }
}

}  // namespace

hipError_t launch_add_norm_rows(int dtype, float *res, const float *y, const int32_t *tokens, const void *embed, float scale, const float *norm_w,
                                float eps, int true_width, void *h, int M, int width, hipStream_t stream) {
    const size_t lds = (size_t)width * sizeof(float);   // (the C ABI keeps width within 64 KiB)
    if (dtype == kF32)
        hipLaunchKernelGGL(add_norm_rows_kernel<float>, dim3(M), dim3(kRowThreads), lds, stream, res, y, tokens, static_cast<const float *>(embed), scale,
                           norm_w, eps, true_width, static_cast<float *>(h), width);
    else
        hipLaunchKernelGGL(add_norm_rows_kernel<bf16>, dim3(M), dim3(kRowThreads), lds, stream, res, y, tokens, static_cast<const bf16 *>(embed), scale, norm_w,
                           eps, true_width, static_cast<bf16 *>(h), width);
    return hipGetLastError();
}

hipError_t launch_embed_rows(int dtype, const int32_t *tokens, const void *embed, float scale, float *res, void *h, int M, int width,
                             hipStream_t stream) {
    if (dtype == kF32)
        hipLaunchKernelGGL(embed_rows_kernel<float>, dim3(M), dim3(kRowThreads), 0, stream, tokens, static_cast<const float *>(embed), scale, res,
                           static_cast<float *>(h), width);
    else
        hipLaunchKernelGGL(embed_rows_kernel<bf16>, dim3(M), dim3(kRowThreads), 0, stream, tokens, static_cast<const bf16 *>(embed), scale, res,
                           static_cast<bf16 *>(h), width);
    return hipGetLastError();
}

hipError_t launch_residual_norm_rows(int dtype, float *res, const void *y, const float *weights, int top, const float *norm_w, float eps,
                                     int true_width, void *h, int M, int width, hipStream_t stream) {
    const size_t lds = (size_t)width * sizeof(float);   // (the C ABI keeps width within 64 KiB)
    if (!weights) top = 0;
    if (dtype == kF32)
        hipLaunchKernelGGL((residual_norm_kernel<float, float>), dim3(M), dim3(kRowThreads), lds, stream, res, static_cast<const float *>(y), weights, top,
                           norm_w, eps, true_width, static_cast<float *>(h), width);
    else if (top > 0)
        hipLaunchKernelGGL((residual_norm_kernel<bf16, bf16>), dim3(M), dim3(kRowThreads), lds, stream, res, static_cast<const bf16 *>(y), weights, top,
                           norm_w, eps, true_width, static_cast<bf16 *>(h), width);
    else
        hipLaunchKernelGGL((residual_norm_kernel<bf16, float>), dim3(M), dim3(kRowThreads), lds, stream, res, static_cast<const float *>(y), weights, top,
                           norm_w, eps, true_width, static_cast<bf16 *>(h), width);
    return hipGetLastError();
}

hipError_t launch_norm_rows(int dtype, const float *res, const int32_t *rows, const float *norm_w, float eps, int true_width, void *out, int n,
                            int width, hipStream_t stream) {
    if (dtype == kF32)
        hipLaunchKernelGGL(norm_rows_kernel<float>, dim3(n), dim3(kRowThreads), 0, stream, res, rows, norm_w, eps, true_width, static_cast<float *>(out),
                           width);
    else
        hipLaunchKernelGGL(norm_rows_kernel<bf16>, dim3(n), dim3(kRowThreads), 0, stream, res, rows, norm_w, eps, true_width, static_cast<bf16 *>(out),
                           width);
    return hipGetLastError();
}

}  // namespace w4a16
