// Mixture of experts behind a grouped sigmoid router, for gfx950.
//
// Choice: score s = sigmoid(logit); choice score s + correction; the experts form `groups` equal groups of neighbours,
// a group counts as much as the sum of its two largest choice scores; the `top` experts with the largest choice scores
// among the `keep` best groups are taken, each with weight s.  Everything in fp32; ties go to the lower index.  One
// wavefront chooses for one token.
//
// One token: the gate / up product makes the choice itself (every workgroup, from the same logits: cheaper than a launch)
// and the first workgroup of a slot leaves it for the down product, which adds the experts' outputs with their weights.
// Many tokens: the choices become (token, slot) entries sorted by expert and cut into row tiles, on which dense_gemm.hip
// runs one grouped product each for gate / up and down.
#include "dense.h"
#include "dense_kernels.h"

namespace w4a16 {

namespace {

constexpr int kMoeWaves = 4, kMoeThreads = 64 * kMoeWaves;
constexpr int kMoePiece = 512;

// Called by one whole wavefront, which owns experts lane + 64 j, j < PL; choice: LDS scratch of r.experts floats, group: of
// r.groups floats (both of this wave).  ids / weights [top] may be LDS or global.
template <int PL>
__device__ __forceinline__ void choose_experts(const Router &r, const float *logits, float *choice, float *group, int32_t *ids,
                                               float *weights) {
    const int lane = threadIdx.x & 63;
    const int size = r.experts / r.groups;
    float score[PL], c[PL];
#pragma unroll
    for (int j = 0; j < PL; ++j) {
        const int e = lane + 64 * j;
        score[j] = 0.f;
        c[j] = -INFINITY;
        if (e < r.experts) {
            score[j] = sigmoid_f32(logits[e]);
            c[j] = score[j] + r.correction[e];
            choice[e] = c[j];
        }
    }
    if (r.groups > 1) {
        __builtin_amdgcn_wave_barrier();
        __threadfence_block();
        for (int g = lane; g < r.groups; g += 64) {
            float a = -INFINITY, b = -INFINITY;   // the two largest
            for (int i = 0; i < size; ++i) {
                const float v = choice[g * size + i];
                b = fmaxf(b, fminf(a, v));
                a = fmaxf(a, v);
            }
            group[g] = size > 1 ? a + b : a;
        }
        __builtin_amdgcn_wave_barrier();
        __threadfence_block();
        // experts outside the kept groups count as minus infinity
#pragma unroll
        for (int j = 0; j < PL; ++j) {
            const int e = lane + 64 * j;
            if (e >= r.experts) continue;
            const int g = e / size;
            const float mine = group[g];
            int better = 0;
            for (int o = 0; o < r.groups; ++o) {
                const float v = group[o];
                better += v > mine || (v == mine && o < g);
            }
            if (better >= r.keep) c[j] = -INFINITY;
        }
    }
    for (int s = 0; s < r.top; ++s) {
        float best = c[0];
#pragma unroll
        for (int j = 1; j < PL; ++j) best = fmaxf(best, c[j]);
        best = wave_reduce<true>(best);
        bool found = false;   // wave-uniform; the lowest index among equals: the first j, its lowest lane
#pragma unroll
        for (int j = 0; j < PL; ++j) {
            const unsigned long long hit = found ? 0ull : __ballot(c[j] == best);
            if (hit) {
                found = true;
                if (lane == __builtin_ctzll(hit)) {
                    ids[s] = lane + 64 * j;
                    weights[s] = score[j];
                    c[j] = -INFINITY;
                }
            }
        }
    }
}

template <class F>
auto with_lanes(int experts, F f) {
    if (experts <= 64) return f(std::integral_constant<int, 1>());
    if (experts <= 256) return f(std::integral_constant<int, 4>());
    return f(std::integral_constant<int, kMaxExperts / 64>());
}

template <int PL>
__global__ void __launch_bounds__(kMoeThreads) moe_select_kernel(const Router r, int tokens, int32_t *ids, float *weights) {
    extern __shared__ float select_lds[];
    const int wave = threadIdx.x >> 6, t = blockIdx.x * kMoeWaves + wave;
    if (t >= tokens) return;   // whole waves leave; no workgroup barrier below
    float *mine = select_lds + wave * (r.experts + r.groups);
    choose_experts<PL>(r, r.logits + (size_t)t * r.ld, mine, mine + r.experts, ids + (size_t)t * r.top, weights + (size_t)t * r.top);
}

// One workgroup: sort the entries by expert (counting sort) and cut every expert's run into tiles of bm entries.
__global__ void __launch_bounds__(1024) moe_plan_kernel(const int32_t *ids, int entries, int experts, int bm, int max_tiles, int32_t *order,
                                                        int32_t *tiles) {
    __shared__ int count[kMaxExperts], first[kMaxExperts], tile0[kMaxExperts + 1], scan[2][1024];
    const int t = threadIdx.x;
    count[t] = 0;   // kMaxExperts == number of threads
    __syncthreads();
    for (int i = t; i < entries; i += 1024) atomicAdd(&count[ids[i]], 1);
    __syncthreads();
    // exclusive prefix sums of the counts and of the tiles per expert
    const int n = count[t];
    for (int what = 0; what < 2; ++what) {
        const int v = what == 0 ? n : (n + bm - 1) / bm;
        int cur = 0;
        scan[0][t] = v;
        __syncthreads();
        for (int d = 1; d < 1024; d *= 2) {
            scan[cur ^ 1][t] = scan[cur][t] + (t >= d ? scan[cur][t - d] : 0);
            cur ^= 1;
            __syncthreads();
        }
        if (what == 0) first[t] = scan[cur][t] - v;
        else {
            tile0[t] = scan[cur][t] - v;
            if (t == 1023) tile0[1024] = scan[cur][t];
        }
        __syncthreads();
    }
    if (t < experts)
        for (int i = 0; i * bm < n; ++i) {
            int32_t *row = tiles + 4 * (tile0[t] + i);
            row[0] = t;
            row[1] = first[t] + i * bm;
            row[2] = n - i * bm < bm ? n - i * bm : bm;
            row[3] = 0;
        }
    if (t == 0) tiles[4 * max_tiles] = tile0[1024];
    count[t] = 0;
    __syncthreads();
    for (int i = t; i < entries; i += 1024) {
        const int e = ids[i];
        order[first[e] + atomicAdd(&count[e], 1)] = i;
    }
}

template <class T>
struct MoeGemv {
    Router r;
    const T *x, *w;
    T *h;
    float *y;
    int32_t *ids;
    float *weights;
    int K, ff, N, top;
};

// h[slot] = silu(gate x) * (up x); blockIdx.y = slot; a wave owns P neighbouring gate rows and the matching up rows
template <class T, int P, int U, int PL>
__global__ void __launch_bounds__(kMoeThreads) moe_gate_up_gemv_kernel(const MoeGemv<T> p) {
    extern __shared__ __attribute__((aligned(16))) char moe_lds[];
    __shared__ int32_t ids[kMaxTop];
    __shared__ float weights[kMaxTop];
    const int kl = (p.K + kMoePiece - 1) / kMoePiece * kMoePiece;
    T *xs = reinterpret_cast<T *>(moe_lds);
    float *scratch = reinterpret_cast<float *>(xs + kl);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, slot = blockIdx.y;
    if (wave == 0) choose_experts<PL>(p.r, p.r.logits, scratch, scratch + p.r.experts, ids, weights);
    else {
        for (int i = 8 * (tid - 64); i < p.K; i += 8 * (kMoeThreads - 64)) store8(xs + i, load8(p.x + i));
        for (int i = p.K + 8 * (tid - 64); i < kl; i += 8 * (kMoeThreads - 64)) store8(xs + i, zero8<T>());
    }
    __syncthreads();
    if (blockIdx.x == 0 && tid == 0) {
        p.ids[slot] = ids[slot];
        p.weights[slot] = weights[slot];
    }
    const T *w = p.w + (size_t)ids[slot] * 2 * p.ff * p.K;
    const int pieces = kl / kMoePiece;
    for (int f0 = (blockIdx.x * kMoeWaves + wave) * P; f0 < p.ff; f0 += gridDim.x * kMoeWaves * P) {
        float g[P], u[P];
#pragma unroll
        for (int j = 0; j < P; ++j) g[j] = u[j] = 0.f;
        // P divides 16, so the P rows lie in one block of 16 gate rows, the up rows 16 further on
        const T *gate = w + (size_t)(f0 / 16 * 32 + f0 % 16) * p.K + 8 * lane, *up = gate + (size_t)16 * p.K;
        for (int c0 = 0; c0 < pieces; c0 += U) {
            Vec8<T> wg[P][U], wu[P][U];
#pragma unroll
            for (int j = 0; j < P; ++j)
#pragma unroll
                for (int c = 0; c < U; ++c) {
                    const int k = (c0 + c) * kMoePiece;
                    const bool in = k + 8 * lane < p.K;
                    wg[j][c] = in ? stream8(gate + (size_t)j * p.K + k) : zero8<T>();
                    wu[j][c] = in ? stream8(up + (size_t)j * p.K + k) : zero8<T>();
                }
#pragma unroll
            for (int c = 0; c < U; ++c) {
                const int pc = c0 + c < pieces ? c0 + c : pieces - 1;
                const Vec8<T> xv = load8(xs + pc * kMoePiece + 8 * lane);
#pragma unroll
                for (int j = 0; j < P; ++j) {
                    g[j] = dot8(wg[j][c], xv, g[j]);
                    u[j] = dot8(wu[j][c], xv, u[j]);
                }
            }
        }
        float mine = 0.f;
#pragma unroll
        for (int j = 0; j < P; ++j) {
            const float v = silu_f32(wave_reduce<false>(g[j])) * wave_reduce<false>(u[j]);
            mine = lane == j ? v : mine;
        }
        if (lane < P) p.h[(size_t)slot * p.ff + f0 + lane] = from_float<T>(mine);
    }
}

// y[n] = sum_s weight_s (down_s h_s)[n]; a wave owns R rows, the pieces of all slots run through one loop
template <class T, int R, int U>
__global__ void __launch_bounds__(kMoeThreads) moe_down_gemv_kernel(const MoeGemv<T> p) {
    extern __shared__ __attribute__((aligned(16))) char moe_lds[];
    T *hs = reinterpret_cast<T *>(moe_lds);
    const int kl = (p.ff + kMoePiece - 1) / kMoePiece * kMoePiece;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    for (int s = 0; s < p.top; ++s) {
        for (int i = 8 * tid; i < p.ff; i += 8 * kMoeThreads) store8(hs + s * kl + i, load8(p.h + (size_t)s * p.ff + i));
        for (int i = p.ff + 8 * tid; i < kl; i += 8 * kMoeThreads) store8(hs + s * kl + i, zero8<T>());
    }
    __syncthreads();
    const int pieces = kl / kMoePiece, items = p.top * pieces;
    for (int n0 = (blockIdx.x * kMoeWaves + wave) * R; n0 < p.N; n0 += gridDim.x * kMoeWaves * R) {
        float acc[R];
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r] = 0.f;
        for (int i0 = 0; i0 < items; i0 += U) {
            Vec8<T> w[R][U];
            float wt[U];
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int i = i0 + u < items ? i0 + u : items - 1;
                const int s = i / pieces, k = (i % pieces) * kMoePiece + 8 * lane;
                wt[u] = i0 + u < items ? p.weights[s] : 0.f;
                const T *base = p.w + (size_t)p.ids[s] * p.N * p.ff + k;
#pragma unroll
                for (int r = 0; r < R; ++r) {
                    const int row = n0 + r < p.N ? n0 + r : p.N - 1;
                    w[r][u] = k < p.ff ? stream8(base + (size_t)row * p.ff) : zero8<T>();
                }
            }
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int i = i0 + u < items ? i0 + u : items - 1;
                const Vec8<T> hv = load8(hs + i * kMoePiece + 8 * lane);   // (slot s, piece c) lies at s * kl + c * 512
#pragma unroll
                for (int r = 0; r < R; ++r) acc[r] = fmaf(wt[u], dot8(w[r][u], hv, 0.f), acc[r]);
            }
        }
        float mine = 0.f;
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const float s = wave_reduce<false>(acc[r]);
            mine = lane == r ? s : mine;
        }
        if (lane < R && n0 + lane < p.N) p.y[n0 + lane] = mine;
    }
}

template <class F>
hipError_t with_lds(F kernel, size_t lds) {
    if (lds <= 48 * 1024) return hipSuccess;
    return hipFuncSetAttribute(reinterpret_cast<const void *>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
}

template <class T>
hipError_t gate_up(const Router &r, const void *x, const void *w, void *h, int32_t *ids, float *weights, int K, int ff, hipStream_t stream) {
    MoeGemv<T> p{};
    p.r = r;
    p.x = static_cast<const T *>(x);
    p.w = static_cast<const T *>(w);
    p.h = static_cast<T *>(h);
    p.ids = ids;
    p.weights = weights;
    p.K = K;
    p.ff = ff;
    p.top = r.top;
    const size_t lds = (size_t)((K + kMoePiece - 1) / kMoePiece) * kMoePiece * sizeof(T) + (size_t)(r.experts + r.groups) * sizeof(float);
    const int P = K > 1024 ? 1 : 2;
    int gx = (ff + kMoeWaves * P - 1) / (kMoeWaves * P);
    const dim3 grid(gx, r.top), block(kMoeThreads);
    auto run = [&](auto kernel) {
        const hipError_t e = with_lds(kernel, lds);
        if (e != hipSuccess) return e;
        hipLaunchKernelGGL(kernel, grid, block, lds, stream, p);
        return hipGetLastError();
    };
    return with_lanes(r.experts, [&](auto pl) {
        constexpr int PL = decltype(pl)::value;
        return P == 1 ? run(&moe_gate_up_gemv_kernel<T, 1, 4, PL>) : run(&moe_gate_up_gemv_kernel<T, 2, 2, PL>);
    });
}

template <class T>
hipError_t down(const void *h, const void *w, const int32_t *ids, const float *weights, float *y, int top, int ff, int N, hipStream_t stream) {
    MoeGemv<T> p{};
    p.h = const_cast<T *>(static_cast<const T *>(h));
    p.w = static_cast<const T *>(w);
    p.ids = const_cast<int32_t *>(ids);
    p.weights = const_cast<float *>(weights);
    p.y = y;
    p.ff = ff;
    p.N = N;
    p.top = top;
    const size_t lds = (size_t)top * ((ff + kMoePiece - 1) / kMoePiece) * kMoePiece * sizeof(T);
    auto kernel = &moe_down_gemv_kernel<T, 1, 8>;
    const hipError_t e = with_lds(kernel, lds);
    if (e != hipSuccess) return e;
    const int need = (N + kMoeWaves - 1) / kMoeWaves;
    hipLaunchKernelGGL(kernel, dim3(need < 1024 ? need : 1024), dim3(kMoeThreads), lds, stream, p);
    return hipGetLastError();
}

}  // namespace

hipError_t launch_moe_gate_up_gemv(int dtype, const Router &r, const void *x, const void *w_gate_up, void *h, int32_t *ids, float *weights, int K,
                                   int ff, hipStream_t stream) {
    return dtype == kF32 ? gate_up<float>(r, x, w_gate_up, h, ids, weights, K, ff, stream)
                         : gate_up<bf16>(r, x, w_gate_up, h, ids, weights, K, ff, stream);
}

hipError_t launch_moe_down_gemv(int dtype, const void *h, const void *w_down, const int32_t *ids, const float *weights, float *y, int top, int ff,
                                int N, hipStream_t stream) {
    return dtype == kF32 ? down<float>(h, w_down, ids, weights, y, top, ff, N, stream) : down<bf16>(h, w_down, ids, weights, y, top, ff, N, stream);
}

hipError_t launch_moe_select(const Router &r, int tokens, int32_t *ids, float *weights, hipStream_t stream) {
    const size_t lds = (size_t)kMoeWaves * (r.experts + r.groups) * sizeof(float);
    return with_lanes(r.experts, [&](auto pl) {
        hipLaunchKernelGGL(moe_select_kernel<decltype(pl)::value>, dim3((tokens + kMoeWaves - 1) / kMoeWaves), dim3(kMoeThreads), lds, stream, r, tokens,
                           ids, weights);
        return hipGetLastError();
    });
}

int moe_max_tiles(int entries, int experts, int bm) { return entries / bm + (entries < experts ? entries : experts); }

hipError_t launch_moe_plan(const int32_t *ids, int entries, int experts, int bm, int32_t *order, int32_t *tiles, hipStream_t stream) {
    hipLaunchKernelGGL(moe_plan_kernel, dim3(1), dim3(1024), 0, stream, ids, entries, experts, bm, moe_max_tiles(entries, experts, bm), order, tiles);
    return hipGetLastError();
}

}  // namespace w4a16
