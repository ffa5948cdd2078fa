// Causal attention of a long portion on expanded keys and values, for gfx950: queries [dim | rot] per head (rotated by
// latent_prepare), keys = the head's dim columns of the expanded matrix followed by the rotated part of the cache row that
// all heads share, values = the head's vdim columns, a learned sink per head in the denominator, and the output gate
// applied before the only store.  WINDOW is the same kernel on grouped keys and values of their own projections
// (head_attention.hip): rows [key | value] of one matrix per key / value head, positions going round in a ring of rows, a limit to
// how far back a query sees, neither sink nor gate.
//
// Both products are computed transposed, so that a lane owns one query from the scores to the output:
//   S^T[key, q] = K . Q^T      A = K rows from LDS, B = Q^T held in registers
//   O^T[d, q]  += V^T . P^T    A = V^T (transposing LDS read), B = P^T built from the lane's own S^T registers
// The D layout gives a lane keys 4 g .. + 3 of each 16-key block; the k slots of the second product are defined as exactly
// those keys, so P never moves between lanes.  Four waves of QB blocks of 16 queries each share the K and V rows going through
// LDS; the next block of keys travels global -> registers while one is multiplied.  With SETS = 2 a second set of four waves
// takes the odd key blocks for the same queries, and the two partial results are merged through LDS at the end: the longest
// rows take half as long, and two waves share a SIMD.  The grid puts the longest rows first.  The running maximum may lag the true one by 2^8 (as in prefill_attention.hip), so
// rescaling is rare; the row sum is a product with a row of ones.
//
// Head sizes that are common have kernels of their own (EXACT: everything unrolled); any other size runs on the next
// larger register allotment with uniform bounds.
#include "dense.h"
#include "dense_kernels.h"

namespace w4a16 {

namespace {

constexpr int kSetThreads = 256;
constexpr float kMasked = -1.0e30f;
constexpr float kNoMax = -1.0e20f;   // "no score yet": far below any score, far above a masked one
constexpr float kLazy = 8.0f;

template <class T>
struct PrefillArgs {
    const T *q, *kv, *cache;
    T *out;
    long ldq, ldkv, ldo;
    int ldc, rot_off;        // cache row length, start of the rotated part in it
    int heads, dim, rot, vdim;
    int v_off, gate_off;     // columns of the values in kv, of the gate in q's matrix
    int M, total;            // queries, keys (the queries are the last M positions)
    float scale_log2;
    const float *sink;
    long head_q, group_q, head_k, head_v;   // elements between two heads' queries, key / value heads' queries, keys, values
    int group, window, ring;                // query heads per key / value head
    float out_scale;
};

template <class T>
__device__ __forceinline__ Vec8<T> ones8();
template <>
__device__ __forceinline__ Vec8<bf16> ones8<bf16>() { return {u32x4{0x3F803F80u, 0x3F803F80u, 0x3F803F80u, 0x3F803F80u}}; }
template <>
__device__ __forceinline__ Vec8<float> ones8<float>() { return {floatx4{1.f, 1.f, 1.f, 1.f}, floatx4{1.f, 1.f, 1.f, 1.f}}; }

// NQ: K-steps of 32 of a score; NV: 16-column tiles of the output; EXACT: the sizes are exactly these, otherwise at most
// these.  blockIdx.z picks a range of 16 NV value columns.
// (EXACT addresses K and V rows with 32-bit offsets: the expanded matrix is smaller than 4 GiB.)
template <class T, int NQ, int NV, int QB, int KB, int SETS, bool EXACT, bool WINDOW>
__global__ void __launch_bounds__(SETS * kSetThreads, SETS) latent_prefill_kernel(const PrefillArgs<T> p) {
    constexpr int NKK = KB / 16, NT = KB / 32, QW = 64 * QB;
    extern __shared__ __attribute__((aligned(16))) char pf_lds[];
    const int tid = threadIdx.x & (kSetThreads - 1), lane = tid & 63;   // thread within its set
    const int wave8 = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int set = SETS == 1 ? 0 : wave8 >> 2, wave = wave8 & 3;
    const int ql = lane & 15, g = lane >> 4;
    const int head = blockIdx.x, item = gridDim.y - 1 - blockIdx.y;
    const int qd = EXACT ? 32 * NQ : p.dim + p.rot;
    const int vcol0 = EXACT ? 0 : blockIdx.z * 16 * NV;
    const int vd = EXACT ? 16 * NV : (p.vdim - vcol0 < 16 * NV ? p.vdim - vcol0 : 16 * NV);
    const int nq = qd / 32, nv = vd / 16;
    const int kp = qd + 16 / (int)sizeof(T), vp = vd + 32 / (int)sizeof(T);
    T *kt = reinterpret_cast<T *>(pf_lds) + set * KB * (kp + vp);
    T *vt = kt + KB * kp;

    const int pos0 = p.total - p.M;
    const int q0 = item * QW + 16 * QB * wave;                    // first query row of this wave
    const int item_end = (item + 1) * QW < p.M ? (item + 1) * QW : p.M;
    const int blocks = (pos0 + item_end + KB - 1) / KB;
    const int wave_last = pos0 + q0 + 16 * QB - 1;                // last position of this wave's queries
    const int kvh = WINDOW ? head / p.group : head;
    // blocks that are wholly in front of the window of every query of the item are left out, and of those of a wave by the wave
    const int item_first = WINDOW ? pos0 + item * QW - p.window + 1 : 0, first = item_first > 0 ? item_first / KB : 0;
    const int wave_first = WINDOW ? pos0 + q0 - p.window + 1 : 0;

    Vec8<T> qf[QB][NQ];
    floatx4 o[QB][NV], l[QB];
    float m[QB];
    int qpos[QB];
#pragma unroll
    for (int b = 0; b < QB; ++b) {
        const int qi = q0 + 16 * b + ql;
        qpos[b] = pos0 + qi;
        const T *row = p.q + (size_t)(qi < p.M ? qi : p.M - 1) * p.ldq + (WINDOW ? kvh * p.group_q + (head - kvh * p.group) * p.head_q : (size_t)head * qd) + 8 * g;
#pragma unroll
        for (int ks = 0; ks < NQ; ++ks)
            if (EXACT || ks < nq) qf[b][ks] = load8(row + 32 * ks);
#pragma unroll
        for (int d = 0; d < NV; ++d) o[b][d] = floatx4{0.f, 0.f, 0.f, 0.f};
        l[b] = floatx4{0.f, 0.f, 0.f, 0.f};
        m[b] = kNoMax;
    }

    // a chunk is 8 elements of a row; the first dim of a K row come from the expanded matrix, the rest from the cache
    const T *k_base = p.kv + kvh * p.head_k, *v_base = p.kv + p.v_off + kvh * p.head_v + vcol0, *r_base = p.cache + p.rot_off;
    auto row_of = [&](int kb, int i) {   // row of key kb + i of a block (a ring holds whole blocks)
        if constexpr (WINDOW) return kb % p.ring + (kb + i < p.total ? i : p.total - 1 - kb);
        const int key = kb + i;
        return key < p.total ? key : p.total - 1;
    };
    auto at = [&](const T *base, int row, long ld, int e) -> Vec8<T> {
        if constexpr (EXACT) return load8(reinterpret_cast<const T *>(reinterpret_cast<const char *>(base) + (uint32_t)(row * (uint32_t)ld + e) * (uint32_t)sizeof(T)));
        return load8(base + (size_t)row * ld + e);
    };
    auto k_chunk = [&](int kb, int c, int cpr) -> Vec8<T> {
        const int row = row_of(kb, c / cpr), e = 8 * (c % cpr);
        return WINDOW || e < p.dim ? at(k_base, row, p.ldkv, e) : at(r_base, row, p.ldc, e - p.dim);
    };
    auto v_chunk = [&](int kb, int c, int cpr) -> Vec8<T> {
        return at(v_base, row_of(kb, c / cpr), p.ldkv, 8 * (c % cpr));
    };
    constexpr int CK = 4 * NQ, CV = 2 * NV;                       // chunks per row (EXACT)
    constexpr int NCK = EXACT ? KB * CK / kSetThreads : 1, NCV = EXACT ? KB * CV / kSetThreads : 1;
    static_assert(!EXACT || (KB * CK % kSetThreads == 0 && KB * CV % kSetThreads == 0), "whole chunks per thread");
    Vec8<T> kreg[NCK], vreg[NCV];
    auto fetch = [&](int it) {
        if constexpr (EXACT) {
#pragma unroll
            for (int i = 0; i < NCK; ++i) kreg[i] = k_chunk(it * KB, tid + kSetThreads * i, CK);
#pragma unroll
            for (int i = 0; i < NCV; ++i) vreg[i] = v_chunk(it * KB, tid + kSetThreads * i, CV);
        }
    };
    auto stage = [&](int it) {
        if constexpr (EXACT) {
#pragma unroll
            for (int i = 0; i < NCK; ++i) {
                const int c = tid + kSetThreads * i;
                store8(kt + (c / CK) * kp + 8 * (c % CK), kreg[i]);
            }
#pragma unroll
            for (int i = 0; i < NCV; ++i) {
                const int c = tid + kSetThreads * i;
                store8(vt + (c / CV) * vp + 8 * (c % CV), vreg[i]);
            }
        } else {
            const int ck = qd / 8, cv = vd / 8;
            for (int c = tid; c < KB * ck; c += kSetThreads) store8(kt + (c / ck) * kp + 8 * (c % ck), k_chunk(it * KB, c, ck));
            for (int c = tid; c < KB * cv; c += kSetThreads) store8(vt + (c / cv) * vp + 8 * (c % cv), v_chunk(it * KB, c, cv));
        }
    };

    if (first + set < blocks) fetch(first + set);
    for (int it0 = first; it0 < blocks; it0 += SETS) {
        const int it = it0 + set, kb = it * KB;
        if (it < blocks) stage(it);
        __syncthreads();
        if (it + SETS < blocks) fetch(it + SETS);
        if (it < blocks && kb <= wave_last && (!WINDOW || kb + KB > wave_first)) {
            floatx4 s[NKK][QB];
#pragma unroll
            for (int kk = 0; kk < NKK; ++kk) {
#pragma unroll
                for (int b = 0; b < QB; ++b) s[kk][b] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int ks = 0; ks < NQ; ++ks)
                    if (EXACT || ks < nq) {
                        const Vec8<T> a = load8(kt + (16 * kk + ql) * kp + 32 * ks + 8 * g);
#pragma unroll
                        for (int b = 0; b < QB; ++b) s[kk][b] = mma32(a, qf[b][ks], s[kk][b]);
                    }
            }
            // s[kk][b][r]: key kb + 16 kk + 4 g + r against query qpos[b]
            const bool masked = kb + KB - 1 > pos0 + q0;
            float bm[QB];
            bool lag = false;
#pragma unroll
            for (int b = 0; b < QB; ++b) {
                if (masked) {
#pragma unroll
                    for (int kk = 0; kk < NKK; ++kk)
#pragma unroll
                        for (int r = 0; r < 4; ++r)
                            if (kb + 16 * kk + 4 * g + r > qpos[b]) s[kk][b][r] = kMasked;
                }
                if (WINDOW && kb <= wave_last - p.window) {
#pragma unroll
                    for (int kk = 0; kk < NKK; ++kk)
#pragma unroll
                        for (int r = 0; r < 4; ++r)
                            if (kb + 16 * kk + 4 * g + r <= qpos[b] - p.window) s[kk][b][r] = kMasked;
                }
                float v = kMasked;
#pragma unroll
                for (int kk = 0; kk < NKK; ++kk) {
                    v = fmaxf(fmaxf(v, s[kk][b][0]), s[kk][b][1]);
                    v = fmaxf(fmaxf(v, s[kk][b][2]), s[kk][b][3]);
                }
                bm[b] = max_over_lane_groups(v);
                lag = lag || (bm[b] - m[b]) * p.scale_log2 > kLazy;
            }
            if (__builtin_amdgcn_ballot_w64(lag) != 0) {   // (always at a query's first visible key)
#pragma unroll
                for (int b = 0; b < QB; ++b) {
                    const float mn = fmaxf(m[b], bm[b]);
                    const float alpha = __builtin_amdgcn_exp2f((m[b] - mn) * p.scale_log2);
                    m[b] = mn;
                    l[b] *= alpha;
#pragma unroll
                    for (int d = 0; d < NV; ++d) o[b][d] *= alpha;
                }
            }
            Vec8<T> pb[QB][NT];
#pragma unroll
            for (int b = 0; b < QB; ++b) {
                const float msc = m[b] * p.scale_log2;
#pragma unroll
                for (int kk = 0; kk < NKK; ++kk)
#pragma unroll
                    for (int r = 0; r < 4; ++r) s[kk][b][r] = __builtin_amdgcn_exp2f(fmaf(s[kk][b][r], p.scale_log2, -msc));
#pragma unroll
                for (int t = 0; t < NT; ++t) {
                    pb[b][t] = pair8<T>(s[2 * t][b], s[2 * t + 1][b]);
                    l[b] = mma32(ones8<T>(), pb[b][t], l[b]);
                }
            }
#pragma unroll
            for (int t = 0; t < NT; ++t)
#pragma unroll
                for (int d = 0; d < NV; ++d)
                    if (EXACT || d < nv) {
                        const Vec8<T> a = column8(vt + 32 * t * vp, vp, 16 * d);
#pragma unroll
                        for (int b = 0; b < QB; ++b) o[b][d] = mma32(a, pb[b][t], o[b][d]);
                    }
        }
        __syncthreads();
    }

    if constexpr (SETS == 2) {   // the same wave and lane of the other set holds the same queries and output elements
        constexpr int NREG = QB * (4 * NV + 2);
        float *xch = reinterpret_cast<float *>(pf_lds) + wave * NREG * 64 + lane;
        if (set == 1) {
#pragma unroll
            for (int b = 0; b < QB; ++b) {
#pragma unroll
                for (int d = 0; d < NV; ++d)
#pragma unroll
                    for (int r = 0; r < 4; ++r) xch[((b * NV + d) * 4 + r) * 64] = o[b][d][r];
                xch[(4 * QB * NV + 2 * b) * 64] = m[b];
                xch[(4 * QB * NV + 2 * b + 1) * 64] = l[b][0];
            }
        }
        __syncthreads();
        if (set == 1) return;
#pragma unroll
        for (int b = 0; b < QB; ++b) {
            const float m1 = xch[(4 * QB * NV + 2 * b) * 64], l1 = xch[(4 * QB * NV + 2 * b + 1) * 64];
            const float mm = fmaxf(m[b], m1);
            const float f0 = __builtin_amdgcn_exp2f((m[b] - mm) * p.scale_log2), f1 = __builtin_amdgcn_exp2f((m1 - mm) * p.scale_log2);
            m[b] = mm;
            l[b][0] = l[b][0] * f0 + l1 * f1;
#pragma unroll
            for (int d = 0; d < NV; ++d)
#pragma unroll
                for (int r = 0; r < 4; ++r) o[b][d][r] = o[b][d][r] * f0 + xch[((b * NV + d) * 4 + r) * 64] * f1;
        }
    }

    const float snk = WINDOW ? 0.f : p.sink[head] * 1.4426950408889634f;
#pragma unroll
    for (int b = 0; b < QB; ++b) {
        const int qi = q0 + 16 * b + ql;
        if (qi >= p.M) continue;
        const float inv = WINDOW ? p.out_scale / l[b][0] : 1.0f / (l[b][0] + exp2f(snk - m[b] * p.scale_log2));
        const int col = head * p.vdim + vcol0 + 4 * g;
        const T *gate = p.q + (size_t)qi * p.ldq + p.gate_off + col;
        T *dst = p.out + (size_t)qi * p.ldo + col;
#pragma unroll
        for (int d = 0; d < NV; ++d)
            if (EXACT || d < nv) {
                float z[4];
                if (!WINDOW) load4(gate + 16 * d, z);
#pragma unroll
                for (int r = 0; r < 4; ++r) z[r] = o[b][d][r] * inv * (WINDOW ? 1.0f : sigmoid_f32(z[r]));
                store4(dst + 16 * d, z[0], z[1], z[2], z[3]);
            }
    }
}

constexpr size_t kLdsLimit = 160 * 1024;

template <class T, int NQ, int NV, int QB, int KB, int SETS, bool EXACT, bool WINDOW = false>
hipError_t launch(const PrefillArgs<T> &p, hipStream_t stream) {
    const int vd = p.vdim < 16 * NV ? p.vdim : 16 * NV;
    size_t lds = (size_t)SETS * KB * ((p.dim + p.rot + 16 / sizeof(T)) + (vd + 32 / sizeof(T))) * sizeof(T);
    const size_t exchange = SETS == 2 ? 4 * QB * (4 * NV + 2) * 64 * sizeof(float) : 0;
    if (lds < exchange) lds = exchange;
    if (lds > kLdsLimit) return hipErrorInvalidValue;
    auto kernel = &latent_prefill_kernel<T, NQ, NV, QB, KB, SETS, EXACT, WINDOW>;
    if (lds > 48 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    const int items = (p.M + 64 * QB - 1) / (64 * QB);
    hipLaunchKernelGGL(kernel, dim3(p.heads, items, (p.vdim + 16 * NV - 1) / (16 * NV)), dim3(SETS * kSetThreads), lds, stream, p);
    return hipGetLastError();
}

template <class T>
PrefillArgs<T> args_of(const LatentShape &s, const LatentRows &r, const void *kv, long ldkv, const float *sink, void *out, long ldo) {
    PrefillArgs<T> p{};
    p.q = static_cast<const T *>(r.proj);
    p.kv = static_cast<const T *>(kv);
    p.cache = static_cast<const T *>(r.cache);
    p.out = static_cast<T *>(out);
    p.ldq = r.ld;
    p.ldkv = ldkv;
    p.ldo = ldo;
    p.ldc = s.rank + s.rot;
    p.rot_off = s.rank;
    p.heads = s.heads;
    p.dim = s.dim;
    p.rot = s.rot;
    p.vdim = s.vdim;
    p.v_off = s.heads * s.dim;
    p.gate_off = r.gate_off;
    p.M = r.M;
    p.total = r.pos + r.M;
    p.scale_log2 = s.scale * 1.4426950408889634f;
    p.sink = sink;
    p.head_k = s.dim;
    p.head_v = s.vdim;
    return p;
}

template <class T>
PrefillArgs<T> args_of(const HeadShape &s, const HeadRows &r, const void *q, void *out, long ldo) {
    PrefillArgs<T> p{};
    p.q = static_cast<const T *>(q);
    p.kv = p.cache = static_cast<const T *>(r.cache);
    p.out = static_cast<T *>(out);
    p.group = s.heads / s.kv_heads;
    p.ldq = (long)p.group * s.dim;
    p.head_q = s.dim;
    p.group_q = (long)r.M * p.ldq;
    p.ldkv = s.dim + s.vdim;
    p.ldo = ldo;
    p.heads = s.heads;
    p.dim = s.dim;
    p.vdim = s.vdim;
    p.v_off = s.dim;
    p.head_k = p.head_v = (long)s.ring * p.ldkv;
    p.window = s.window;
    p.ring = s.ring;
    p.M = r.M;
    p.total = r.pos + r.M;
    p.scale_log2 = s.scale * 1.4426950408889634f;
    p.out_scale = s.out_scale;
    return p;
}

}  // namespace

bool latent_prefill_supported(int dtype, const LatentShape &s) {
    (void)dtype;
    return s.dim + s.rot <= 512;
}

hipError_t launch_latent_prefill(int dtype, const LatentShape &s, const LatentRows &r, const void *kv, long ldkv, const float *sink, void *out,
                                 long ldo, hipStream_t stream) {
    const int nq = (s.dim + s.rot) / 32, nv = s.vdim / 16;
    if (dtype == kF32) {
        const PrefillArgs<float> p = args_of<float>(s, r, kv, ldkv, sink, out, ldo);
        if (nq <= 4 && nv <= 4) return launch<float, 4, 4, 1, 32, 1, false>(p, stream);
        if (nq <= 8 && nv <= 8) return launch<float, 8, 8, 1, 32, 1, false>(p, stream);
        return launch<float, 16, 16, 1, 32, 1, false>(p, stream);
    }
    const PrefillArgs<bf16> p = args_of<bf16>(s, r, kv, ldkv, sink, out, ldo);
    if ((double)p.total * ldkv * sizeof(bf16) < 4e9) {
        if (nq == 6 && nv == 8) return launch<bf16, 6, 8, 2, 64, 2, true>(p, stream);
        if (nq == 3 && nv == 4) return launch<bf16, 3, 4, 2, 64, 2, true>(p, stream);
    }
    if (nq <= 4 && nv <= 4) return launch<bf16, 4, 4, 1, 64, 1, false>(p, stream);
    if (nq <= 8 && nv <= 8) return launch<bf16, 8, 8, 1, 64, 1, false>(p, stream);
    return launch<bf16, 16, 16, 1, 32, 1, false>(p, stream);
}

bool head_prefill_supported(int dtype, const HeadShape &s) {
    (void)dtype;
    return s.dim <= 512;
}

hipError_t launch_head_prefill(int dtype, const HeadShape &s, const HeadRows &r, const void *q, void *out, long ldo, hipStream_t stream) {
    const int nq = s.dim / 32, nv = s.vdim / 16;
    if (dtype == kF32) {
        const PrefillArgs<float> p = args_of<float>(s, r, q, out, ldo);
        if (nq <= 4 && nv <= 4) return launch<float, 4, 4, 1, 32, 1, false, true>(p, stream);
        if (nq <= 8 && nv <= 8) return launch<float, 8, 8, 1, 32, 1, false, true>(p, stream);
        return launch<float, 16, 16, 1, 32, 1, false, true>(p, stream);
    }
    const PrefillArgs<bf16> p = args_of<bf16>(s, r, q, out, ldo);
    if ((double)s.ring * (s.dim + s.vdim) * sizeof(bf16) < 4e9) {
        if (nq == 4 && nv == 8) return launch<bf16, 4, 8, 2, 64, 2, true, true>(p, stream);
        if (nq == 2 && nv == 4) return launch<bf16, 2, 4, 2, 64, 2, true, true>(p, stream);
    }
    if (nq <= 4 && nv <= 4) return launch<bf16, 4, 4, 1, 64, 1, false, true>(p, stream);
    if (nq <= 8 && nv <= 8) return launch<bf16, 8, 8, 1, 64, 1, false, true>(p, stream);
    return launch<bf16, 16, 16, 1, 32, 1, false, true>(p, stream);
}

}  // namespace w4a16
