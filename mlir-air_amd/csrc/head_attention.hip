// Windowed attention of grouped heads for gfx950: what stands in front of and behind the two attention kernels, which are those of
// the latent attention (latent_attention.hip for few rows, latent_prefill.hip for many) on another view of the cache.
//
//   head_prepare   the norms of the queries and keys (RMS over a head, one weight for all heads), the queries in the order the
//                  kernels read, the cache rows [normed key | value] appended at position % ring
//   head_merge     the splits of the keys merged
#include "dense.h"
#include "dense_kernels.h"

namespace w4a16 {

namespace {

constexpr int kPrepThreads = 256;

// Vectors of one head by groups of `lanes` lanes, eight elements per lane at a time.
__host__ __device__ inline int lanes_of(int n) {
    int l = 1;
    while (l < 64 && 8 * l < n) l *= 2;
    return l;
}

// blockIdx.y = token; blockIdx.x: vectors of the token (queries, keys, values), 256 / lanes at a time
template <class T>
__global__ void __launch_bounds__(kPrepThreads) head_prepare_kernel(const HeadShape s, const T *proj, long ld, const float *q_norm, const float *k_norm,
                                                                    float eps, T *cache, int M, const int32_t *pos_dev, int pos, T *q, int lanes) {
    const int m = blockIdx.y, position = (pos_dev ? pos_dev[0] : pos) + m;
    const int lane = threadIdx.x % lanes, unit = blockIdx.x * (kPrepThreads / lanes) + threadIdx.x / lanes;
    const int H = s.heads, G = s.kv_heads, group = H / G, row_len = s.dim + s.vdim;
    if (unit >= H + 2 * G) return;
    const bool is_q = unit < H, is_v = unit >= H + G;
    const T *src = proj + (size_t)m * ld + (is_v ? (size_t)(H + G) * s.dim + (size_t)(unit - H - G) * s.vdim : (size_t)unit * s.dim);
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
        rstd = 1.0f / sqrtf(group_sum(ss, lanes) / (float)s.true_dim + eps);
    }
    const float *w = is_q ? q_norm : k_norm;
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

constexpr int kMergeThreads = 256, kMaxSplits = 256;

// blockIdx.x = query head, blockIdx.y = token
template <class T>
__global__ void __launch_bounds__(kMergeThreads) head_merge_kernel(const HeadShape s, int M, const int32_t *pos_dev, int pos, int nsplit, int kb,
                                                                   const float *part_o, const float *part_ml, T *out, long ldo) {
    __shared__ float f[kMaxSplits];
    __shared__ float red[8];
    __shared__ floatx4 part[kMergeThreads];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int group = s.heads / s.kv_heads, h = blockIdx.x, m = blockIdx.y;
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
    for (int c0 = 0; c0 < s.vdim; c0 += 4 * kMergeThreads) {
        const int width = (s.vdim - c0) / 4 < kMergeThreads ? (s.vdim - c0) / 4 : kMergeThreads;   // four-column pieces of this round
        const int ways = kMergeThreads / width, way = tid / width, col = c0 + 4 * (tid % width);
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
    const int lanes = lanes_of(s.dim > s.vdim ? s.dim : s.vdim), per = kPrepThreads / lanes;
    const dim3 grid((s.heads + 2 * s.kv_heads + per - 1) / per, r.M);
    if (dtype == kF32)
        hipLaunchKernelGGL(head_prepare_kernel<float>, grid, dim3(kPrepThreads), 0, stream, s, static_cast<const float *>(r.proj) + r.off, r.ld, r.q_norm,
                           r.k_norm, r.eps, static_cast<float *>(r.cache), r.M, r.pos_dev, r.pos, static_cast<float *>(q), lanes);
    else
        hipLaunchKernelGGL(head_prepare_kernel<bf16>, grid, dim3(kPrepThreads), 0, stream, s, static_cast<const bf16 *>(r.proj) + r.off, r.ld, r.q_norm,
                           r.k_norm, r.eps, static_cast<bf16 *>(r.cache), r.M, r.pos_dev, r.pos, static_cast<bf16 *>(q), lanes);
    return hipGetLastError();
}

hipError_t launch_head_merge(int dtype, const HeadShape &s, const HeadRows &r, int nsplit, const float *part_o, const float *part_ml, void *out, long ldo,
                             hipStream_t stream) {
    const int kb = decode_block_keys(dtype, head_view(s));
    const dim3 grid(s.heads, r.M);
    if (dtype == kF32)
        hipLaunchKernelGGL(head_merge_kernel<float>, grid, dim3(kMergeThreads), 0, stream, s, r.M, r.pos_dev, r.pos, nsplit, kb, part_o, part_ml,
                           static_cast<float *>(out), ldo);
    else
        hipLaunchKernelGGL(head_merge_kernel<bf16>, grid, dim3(kMergeThreads), 0, stream, s, r.M, r.pos_dev, r.pos, nsplit, kb, part_o, part_ml,
                           static_cast<bf16 *>(out), ldo);
    return hipGetLastError();
}

}  // namespace w4a16
