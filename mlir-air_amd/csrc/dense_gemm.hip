// Products over many rows with dense weights for gfx950: out[M, N] = A[M, K] W[N, K]^T, A and W row-major in the element
// type, fp32 accumulation; plain, or grouped over the experts of a mixture (row tiles from moe_plan_kernel).
//
// Both operands have k contiguous, so a tile of either is a set of rows of 128 bytes per K-step (64 bf16 or 32 floats) and
// goes global -> LDS without passing through registers (global_load_lds_dwordx4) into a ring of STAGES buffers, STAGES - 1
// K-steps ahead (two where the tile is large; the small tile has little to multiply per step): one wave instruction
// fills 1 KiB, 8 rows, lane l writing 16-byte slot l % 8 of row l / 8 and fetching chunk slot ^ row % 8, so that the operand
// reads of 16 consecutive rows are spread over the banks without padding.  One barrier per K-step.  W is the first MFMA
// operand: a lane then holds four consecutive n of one row m and stores them as one word.
//
// Row gathers cost nothing here: every lane of a copy has its own source row.  The waves of a SIMD differ in their rows, so
// that a wave whose rows lie behind the end of an expert's run can leave the matrix pipe to the other.
//
// Requirements: K a multiple of 128 bytes of elements (the loader pads), N of 16.  Rows past M and N are read from the last
// row and never stored.
#include "dense.h"
#include "dense_kernels.h"

namespace w4a16 {

namespace {

constexpr int kRowBytes = 128;

template <class T>
struct GemmKernelArgs {
    const T *a, *w;
    void *out;
    int M, N, K;
    long lda, ldo;
    const int32_t *tiles, *order;
    int gather;
    long w_stride;
    int tiles_m, tiles_n;
    int silu_begin, silu_end;
};

// BM x BN tile, WM x WN waves (m x n); GROUPED: expert row tiles
template <class T, int BM, int BN, int WM, int WN, int STAGES, int EPI, bool GROUPED>
__global__ void __launch_bounds__(64 * WM * WN) dense_gemm_kernel(const GemmKernelArgs<T> p) {
    constexpr int NW = WM * WN, KE = kRowBytes / sizeof(T), KS = KE / 32;
    constexpr int MT = BM / WM / 16, NT = BN / WN / 16;
    constexpr int COPIES = (BM + BN) / 8 / NW;
    static_assert((BM + BN) % (8 * NW) == 0, "whole copies per wave");
    constexpr int kStage = (BM + BN) * kRowBytes;
    extern __shared__ __attribute__((aligned(16))) char gemm_lds[];

    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wm = wave / WN, wn = wave % WN;
    const int ql = lane & 15, g = lane >> 4;

    // An XCD (blockIdx % 8) takes a contiguous range of tiles; in a band of four row panels the columns go by first, so
    // that the workgroups running together on one XCD share both operands in its L2.
    // (Experts: the launch covers the most tiles that there can be, the table's last row says how many there are.)
    const int tiles_m = GROUPED ? p.tiles[4 * p.tiles_m] : p.tiles_m;
    const int total = tiles_m * p.tiles_n, per_xcd = (total + 7) / 8;
    const int tile = (blockIdx.x & 7) * per_xcd + (blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= per_xcd || tile >= total) return;
    const int band = tile / (4 * p.tiles_n), in_band = tile % (4 * p.tiles_n);
    const int rows_in_band = tiles_m - 4 * band < 4 ? tiles_m - 4 * band : 4;
    const int tm = 4 * band + in_band % rows_in_band, tn = in_band / rows_in_band;

    const T *w = p.w;
    int m0 = tm * BM, m_end = p.M;
    if constexpr (GROUPED) {
        const int32_t *t = p.tiles + 4 * tm;
        w += (size_t)t[0] * p.w_stride;
        m0 = t[1];
        m_end = m0 + t[2];
    }
    const int n0 = tn * BN;

    // copy sources of this lane: row (lane / 8) of the eight rows of copy i, chunk (lane % 8) ^ row % 8
    const char *src[COPIES];
#pragma unroll
    for (int i = 0; i < COPIES; ++i) {
        const int row = 8 * (i * NW + wave) + (lane >> 3);   // row of the stage: A rows, then W rows
        const T *base;
        if (row < BM) {
            int m = m0 + row < m_end ? m0 + row : m_end - 1;
            if constexpr (GROUPED)
                if (p.gather > 0) m = p.order[m] / p.gather;
            base = p.a + (size_t)m * p.lda;
        } else {
            const int n = n0 + row - BM < p.N ? n0 + row - BM : p.N - 1;
            base = w + (size_t)n * p.K;
        }
        src[i] = reinterpret_cast<const char *>(base) + 16 * ((lane & 7) ^ (row & 7));
    }
    auto copy = [&](int buf, int kt) {
#pragma unroll
        for (int i = 0; i < COPIES; ++i)
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void *)(src[i] + (size_t)kt * kRowBytes),
                                             (__attribute__((address_space(3))) void *)(gemm_lds + buf * kStage + 1024 * (i * NW + wave)), 16, 0, 0);
    };
    auto operand = [&](const char *stage, int row, int ks) -> Vec8<T> {   // 8 consecutive k of a stage row
        const char *r = stage + row * kRowBytes;
        if constexpr (sizeof(T) == 2) {
            return load8(reinterpret_cast<const T *>(r + 16 * ((4 * ks + g) ^ (row & 7))));
        } else {
            Vec8<T> v;
            v.lo = *reinterpret_cast<const floatx4 *>(r + 16 * ((2 * g) ^ (row & 7)));
            v.hi = *reinterpret_cast<const floatx4 *>(r + 16 * ((2 * g + 1) ^ (row & 7)));
            return v;
        }
    };

    floatx4 acc[NT][MT];
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
        for (int i = 0; i < MT; ++i) acc[j][i] = floatx4{0.f, 0.f, 0.f, 0.f};

    const int steps = p.K / KE;
    const bool idle = GROUPED && m0 + wm * (BM / WM) >= m_end;
#pragma unroll
    for (int i = 0; i < STAGES - 1; ++i)
        if (i < steps) copy(i, i);
    int buf = 0;
    for (int kt = 0; kt < steps; ++kt) {
        // The copies write LDS behind the compiler's back: step kt's have landed once at most those of the STAGES - 2 steps
        // after it are outstanding; this wave's reads of the step before have returned.  Then, behind the barrier, so have
        // everybody's, and the buffer of the step before can be filled again.
        if (STAGES > 2 && kt + STAGES - 2 < steps) asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" ::"n"((STAGES - 2) * COPIES) : "memory");
        else asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();
        asm volatile("" ::: "memory");
        const int next = buf == 0 ? STAGES - 1 : buf - 1;   // the buffer of the step before = of the step STAGES - 1 ahead
        if (kt + STAGES - 1 < steps) copy(next, kt + STAGES - 1);
        const char *stage = gemm_lds + buf * kStage;
        buf = buf + 1 == STAGES ? 0 : buf + 1;
        if (idle) continue;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            Vec8<T> b[MT], a[NT];
#pragma unroll
            for (int i = 0; i < MT; ++i) b[i] = operand(stage, wm * (BM / WM) + 16 * i + ql, ks);
#pragma unroll
            for (int j = 0; j < NT; ++j) a[j] = operand(stage, BM + wn * (BN / WN) + 16 * j + ql, ks);
#pragma unroll
            for (int j = 0; j < NT; ++j)
#pragma unroll
                for (int i = 0; i < MT; ++i) acc[j][i] = mma32(a[j], b[i], acc[j][i]);
        }
    }

    // lane: row m = ... + ql, columns 4 g .. + 3 of each 16-column block
#pragma unroll
    for (int i = 0; i < MT; ++i) {
        const int m = m0 + wm * (BM / WM) + 16 * i + ql;
        if (m >= m_end) continue;
        size_t row = m;
        if constexpr (GROUPED)
            if (p.gather == 0) row = p.order[m];
        if constexpr (EPI == kOutSwiglu || EPI == kOutGeglu) {
#pragma unroll
            for (int j = 0; j < NT; j += 2) {
                const int n = n0 + wn * (BN / WN) + 16 * j;
                if (n >= p.N) continue;
                float v[4];
#pragma unroll
                for (int r = 0; r < 4; ++r) v[r] = (EPI == kOutGeglu ? gelu_tanh_f32(acc[j][i][r]) : silu_f32(acc[j][i][r])) * acc[j + 1][i][r];
                store4(static_cast<T *>(p.out) + row * p.ldo + n / 2 + 4 * g, v[0], v[1], v[2], v[3]);
            }
        } else {
#pragma unroll
            for (int j = 0; j < NT; ++j) {
                const int n = n0 + wn * (BN / WN) + 16 * j + 4 * g;
                if (n >= p.N) continue;
                if constexpr (EPI == kOutElem && !GROUPED) {
                    if (n >= p.silu_begin && n < p.silu_end) {
#pragma unroll
                        for (int r = 0; r < 4; ++r) acc[j][i][r] = silu_f32(acc[j][i][r]);
                    }
                }
                if constexpr (EPI == kOutF32)
                    store4(static_cast<float *>(p.out) + row * p.ldo + n, acc[j][i][0], acc[j][i][1], acc[j][i][2], acc[j][i][3]);
                else
                    store4(static_cast<T *>(p.out) + row * p.ldo + n, acc[j][i][0], acc[j][i][1], acc[j][i][2], acc[j][i][3]);
            }
        }
    }
}

template <class T, int BM, int BN, int WM, int WN, int STAGES>
hipError_t launch_tile(const GemmArgs &g, hipStream_t stream) {
    GemmKernelArgs<T> p;
    p.a = static_cast<const T *>(g.a);
    p.w = static_cast<const T *>(g.w);
    p.out = g.out;
    p.M = g.M;
    p.N = g.N;
    p.K = g.K;
    p.lda = g.lda;
    p.ldo = g.ldo;
    p.tiles = g.tiles;
    p.order = g.order;
    p.gather = g.gather;
    p.w_stride = g.w_stride;
    p.silu_begin = g.silu_begin;
    p.silu_end = g.silu_end;
    p.tiles_m = g.tiles ? g.n_tiles : (g.M + BM - 1) / BM;
    p.tiles_n = (g.N + BN - 1) / BN;
    const int total = p.tiles_m * p.tiles_n, grid = (total + 7) / 8 * 8;
    constexpr size_t lds = STAGES * (size_t)(BM + BN) * kRowBytes;
    auto run = [&](auto kernel) {
        if (lds > 48 * 1024) {
            const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
            if (e != hipSuccess) return e;
        }
        hipLaunchKernelGGL(kernel, dim3(grid), dim3(64 * WM * WN), lds, stream, p);
        return hipGetLastError();
    };
    if (g.tiles)
        return g.epilogue == kOutSwiglu ? run(&dense_gemm_kernel<T, BM, BN, WM, WN, STAGES, kOutSwiglu, true>)
                                        : run(&dense_gemm_kernel<T, BM, BN, WM, WN, STAGES, kOutElem, true>);
    switch (g.epilogue) {
        case kOutF32: return run(&dense_gemm_kernel<T, BM, BN, WM, WN, STAGES, kOutF32, false>);
        case kOutSwiglu: return run(&dense_gemm_kernel<T, BM, BN, WM, WN, STAGES, kOutSwiglu, false>);
        case kOutGeglu: return run(&dense_gemm_kernel<T, BM, BN, WM, WN, STAGES, kOutGeglu, false>);
        default: return run(&dense_gemm_kernel<T, BM, BN, WM, WN, STAGES, kOutElem, false>);
    }
}

}  // namespace

// Rows of A per tile for a product of `rows` rows with each of `matrices` matrices.  Measured: full of work, the 256 x 256
// kernel runs at 1.22 PFLOP/s with one workgroup per CU, the 128 x 128 one at 0.9 to 1.0 with two; each loses what its last
// round of workgroups leaves idle.  Experts with enough rows take the large tile (their tiles are rarely full in either case).
int dense_gemm_tile_rows(int dtype, int rows, int N, int matrices) {
    if (rows <= 48 || N < 96) return 32;
    if (dtype != kBf16) return 128;
    if (matrices > 1) return rows >= 160 && N >= 256 ? 256 : 128;
    const int t256 = ((rows + 255) / 256) * ((N + 255) / 256), t128 = ((rows + 127) / 128) * ((N + 127) / 128);
    const float e256 = 1.22f * t256 / ((t256 + 255) / 256 * 256);
    const float e128 = t128 < 512 ? 1.1f * t128 / 512 : 0.88f * t128 / ((t128 + 255) / 256 * 256);
    return e256 > e128 ? 256 : 128;
}

hipError_t launch_dense_gemm(int dtype, const GemmArgs &g, int tile_rows, hipStream_t stream) {
    if (dtype == kF32) return tile_rows == 32 ? launch_tile<float, 32, 128, 1, 4, 4>(g, stream) : launch_tile<float, 128, 128, 2, 2, 2>(g, stream);
    switch (tile_rows) {
        case 32: return launch_tile<bf16, 32, 128, 1, 4, 4>(g, stream);
        case 128: return launch_tile<bf16, 128, 128, 2, 2, 2>(g, stream);
        default: return launch_tile<bf16, 256, 256, 2, 4, 2>(g, stream);
    }
}

}  // namespace w4a16
