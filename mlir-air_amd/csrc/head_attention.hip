// Windowed attention of grouped heads for gfx950: what stands in front of and behind the two attention kernels, which are those of
// the latent attention (latent_attention.hip for few rows, latent_prefill.hip for many) on another view of the cache.
//
//   head_prepare   the norms of the queries and keys (RMS over a head, one weight for all heads), the queries in the order the
//                  kernels read, the cache rows [normed key | value] appended at position % ring
//   head_merge     the splits of the keys merged
#include "dense.h"
#include "dense_kernels.h"
#include "mixer_steps.h"

namespace w4a16 {

namespace {

// blockIdx.y = token
template <class T>
__global__ void __launch_bounds__(kStepThreads) head_prepare_kernel(const HeadShape s, const HeadRows r, T *q, int lanes) {
    head_prepare_step<T>(s, r, q, lanes, blockIdx.x, blockIdx.y);
}

// blockIdx.x = query head, blockIdx.y = token
template <class T>
__global__ void __launch_bounds__(kStepThreads) head_merge_kernel(const HeadShape s, int M, const int32_t *pos_dev, int pos, int nsplit, int kb,
                                                                  const float *part_o, const float *part_ml, T *out, long ldo) {
    __shared__ float f[kMergeSplits];
    __shared__ float red[8];
    __shared__ floatx4 part[kStepThreads];
    head_merge_step<T>(s, M, pos_dev, pos, nsplit, kb, part_o, part_ml, out, ldo, blockIdx.x, blockIdx.y, f, red, part);
}

}  // namespace

CacheView head_view(const HeadShape &s) {
    CacheView v;
    v.heads = s.heads / s.kv_heads;
    v.kv_heads = s.kv_heads;
    v.q_len = s.dim;
    v.row_len = s.dim + s.vdim;
    v.v_off = s.dim;
    v.v_cols = s.vdim;
    v.window = s.window;
    v.ring = s.ring;
    v.head_stride = (long)s.ring * v.row_len;
    v.scale = s.scale;
    return v;
}

hipError_t launch_head_prepare(int dtype, const HeadShape &s, const HeadRows &r, void *q, hipStream_t stream) {
    const int lanes = lanes_of(s.dim > s.vdim ? s.dim : s.vdim, 8), per = kStepThreads / lanes;
    const dim3 grid((s.heads + 2 * s.kv_heads + per - 1) / per, r.M);
    if (dtype == kF32) hipLaunchKernelGGL(head_prepare_kernel<float>, grid, dim3(kStepThreads), 0, stream, s, r, static_cast<float *>(q), lanes);
    else hipLaunchKernelGGL(head_prepare_kernel<bf16>, grid, dim3(kStepThreads), 0, stream, s, r, static_cast<bf16 *>(q), lanes);
    return hipGetLastError();
}

hipError_t launch_head_merge(int dtype, const HeadShape &s, const HeadRows &r, int nsplit, const float *part_o, const float *part_ml, void *out, long ldo,
                             hipStream_t stream) {
    const int kb = decode_block_keys(dtype, head_view(s));
    const dim3 grid(s.heads, r.M);
    if (dtype == kF32)
        hipLaunchKernelGGL(head_merge_kernel<float>, grid, dim3(kStepThreads), 0, stream, s, r.M, r.pos_dev, r.pos, nsplit, kb, part_o, part_ml,
                           static_cast<float *>(out), ldo);
    else
        hipLaunchKernelGGL(head_merge_kernel<bf16>, grid, dim3(kStepThreads), 0, stream, s, r.M, r.pos_dev, r.pos, nsplit, kb, part_o, part_ml,
                           static_cast<bf16 *>(out), ldo);
    return hipGetLastError();
}

}  // namespace w4a16
