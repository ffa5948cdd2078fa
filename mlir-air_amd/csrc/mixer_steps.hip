// Steps of one token that do not wait for each other, sharing a launch: the workgroups of the first follow those of the second.
//
//   head_state_begin   norm of the queries and keys + cache append (head_attention.hip)  |  state step with a decay per head
//   head_state_end     merge of the split keys                                           |  norm and gate of the read-outs
//   conv_products      short convolution                                                 |  two products of short rows
#include "dense.h"
#include "dense_kernels.h"
#include "mixer_steps.h"

namespace w4a16 {

namespace {

template <class T, int ND>
__global__ void __launch_bounds__(kStepThreads) head_state_begin_kernel(const HeadShape s, const HeadRows r, T *q, int lanes, int head_blocks,
                                                                        const LinearArgs a, float *o) {
    const int tiles = a.vdim / 16, step_blocks = a.heads * tiles;
    if ((int)blockIdx.x < step_blocks) recurrence_step<T, ND, false>(a, o, blockIdx.x / tiles, blockIdx.x % tiles);
    else head_prepare_step<T>(s, r, q, lanes, blockIdx.x - step_blocks, 0);
}

template <class T>
__global__ void __launch_bounds__(kStepThreads) head_state_end_kernel(const HeadShape s, const int32_t *pos_dev, int pos, int nsplit, int kb, const float *part_o,
                                                                      const float *part_ml, T *out, const GatedNorm g, const T *gate, T *norm_out) {
    __shared__ float f[kMergeSplits];
    __shared__ float red[8];
    __shared__ floatx4 part[kStepThreads];
    if (blockIdx.x == 0) gated_norm_row_step<T>(g, gate, norm_out, 0, red);
    else head_merge_step<T>(s, 1, pos_dev, pos, nsplit, kb, part_o, part_ml, out, 0, blockIdx.x - 1, 0, f, red, part);
}

template <class T>
__global__ void __launch_bounds__(kStepThreads) conv_products_kernel(const ConvArgs c, const T *proj, T *history, T *act, int lanes, int conv_blocks,
                                                                     const ShortRows<T, float> a, const ShortRows<T, T> b) {
    int block = blockIdx.x;
    if (block < conv_blocks) {
        short_conv_step<T>(c, proj, history, act, lanes, block, 0);
        return;
    }
    block -= conv_blocks;
    if (block < a.blocks) short_rows_step<T, float>(a.w, a.x, a.K, a.N, a.out, a.lanes, block);
    else short_rows_step<T, T>(b.w, b.x, b.K, b.N, b.out, b.lanes, block - a.blocks);
}

template <class T, class O>
ShortRows<T, O> short_rows(const ShortProduct &p) {
    ShortRows<T, O> r;
    r.w = static_cast<const T *>(p.w);
    r.x = static_cast<const T *>(p.x);
    r.out = static_cast<O *>(p.out);
    r.K = p.K;
    r.N = p.N;
    r.lanes = lanes_of(p.K, 8);
    const int per = kStepThreads / r.lanes * kRowsAtOnce;
    r.blocks = (p.N + per - 1) / per;
    return r;
}

template <class T>
hipError_t begin(const HeadShape &s, const HeadRows &r, void *q, const LinearArgs &a, float *o, hipStream_t stream) {
    const int lanes = lanes_of(s.dim > s.vdim ? s.dim : s.vdim, 8), per = kStepThreads / lanes;
    const int head_blocks = (s.heads + 2 * s.kv_heads + per - 1) / per, step_blocks = a.heads * (a.vdim / 16);
    auto run = [&](auto kernel) {
        hipLaunchKernelGGL(kernel, dim3(head_blocks + step_blocks), dim3(kStepThreads), 0, stream, s, r, static_cast<T *>(q), lanes, head_blocks, a, o);
        return hipGetLastError();
    };
    switch (a.dim / 64) {
        case 1: return run(&head_state_begin_kernel<T, 1>);
        case 2: return run(&head_state_begin_kernel<T, 2>);
        case 3: return run(&head_state_begin_kernel<T, 3>);
        case 4: return run(&head_state_begin_kernel<T, 4>);
        case 5: return run(&head_state_begin_kernel<T, 5>);
        case 6: return run(&head_state_begin_kernel<T, 6>);
        case 7: return run(&head_state_begin_kernel<T, 7>);
        case 8: return run(&head_state_begin_kernel<T, 8>);
        default: return hipErrorInvalidValue;
    }
}

template <class T>
hipError_t end(int dtype, const HeadShape &s, const HeadRows &r, int nsplit, const float *part_o, const float *part_ml, void *out, const GatedNorm &g,
               const void *gate, void *norm_out, hipStream_t stream) {
    hipLaunchKernelGGL(head_state_end_kernel<T>, dim3(1 + s.heads), dim3(kStepThreads), 0, stream, s, r.pos_dev, r.pos, nsplit,
                       decode_block_keys(dtype, head_view(s)), part_o, part_ml, static_cast<T *>(out), g, static_cast<const T *>(gate), static_cast<T *>(norm_out));
    return hipGetLastError();
}

template <class T>
hipError_t conv_products(const ConvArgs &c, const void *proj, void *history, void *act, const ShortProduct &pa, const ShortProduct &pb, hipStream_t stream) {
    const int lanes = lanes_of(c.dim > c.vdim ? c.dim : c.vdim, 8), per = kStepThreads / lanes;
    const int conv_blocks = (2 * c.k_heads + c.heads + per - 1) / per;
    const ShortRows<T, float> a = short_rows<T, float>(pa);
    const ShortRows<T, T> b = short_rows<T, T>(pb);
    hipLaunchKernelGGL(conv_products_kernel<T>, dim3(conv_blocks + a.blocks + b.blocks), dim3(kStepThreads), 0, stream, c, static_cast<const T *>(proj) + c.off,
                       static_cast<T *>(history), static_cast<T *>(act), lanes, conv_blocks, a, b);
    return hipGetLastError();
}

}  // namespace

hipError_t launch_head_state_begin(int dtype, const HeadShape &s, const HeadRows &r, void *q, const LinearArgs &a, float *o, hipStream_t stream) {
    return dtype == kF32 ? begin<float>(s, r, q, a, o, stream) : begin<bf16>(s, r, q, a, o, stream);
}

hipError_t launch_head_state_end(int dtype, const HeadShape &s, const HeadRows &r, int nsplit, const float *part_o, const float *part_ml, void *out,
                                 const GatedNorm &g, const void *gate, void *norm_out, hipStream_t stream) {
    return dtype == kF32 ? end<float>(dtype, s, r, nsplit, part_o, part_ml, out, g, gate, norm_out, stream)
                         : end<bf16>(dtype, s, r, nsplit, part_o, part_ml, out, g, gate, norm_out, stream);
}

hipError_t launch_conv_products(int dtype, const ConvArgs &c, const void *proj, void *history, void *act, const ShortProduct &a, const ShortProduct &b,
                                hipStream_t stream) {
    return dtype == kF32 ? conv_products<float>(c, proj, history, act, a, b, stream) : conv_products<bf16>(c, proj, history, act, a, b, stream);
}

}  // namespace w4a16
