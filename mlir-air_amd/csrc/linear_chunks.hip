// Linear recurrences over long portions for gfx950, in chunks of 64 tokens (see linear_attention.hip for the recurrence).
//
// Within a chunk, with G_i the sum of the log decays of tokens 0 .. i of the chunk (per head or per key channel), S the state in
// front of it and <a, b>_G products whose channels are weighted:
//
//   A_ij = <k_i, k_j e^(G_i - G_j)>  (j < i),   B_ij = <q_i, k_j e^(G_i - G_j)>  (j <= i)
//   (1 + diag(beta) A) U = diag(beta) (V - (k e^G) S)       u of the delta rule; U = V without it
//   O = (q e^G) S + B U,    S' = e^(G_last) S + (k e^(G_last - G))^T U
//
// so that everything but the products with S can be done for all chunks at once:
//
//   linear_chunk / delta_chunk   one workgroup per head and chunk: q e^G, (k e^(G_last - G))^T, B, e^(G_last), and U as
//                                U0 - W S: U0 = V, or U0 = (1 + diag(beta) A)^-1 diag(beta) V and W the same of k e^G
//   chunk_scan                   one workgroup per head and 16 value columns goes through the chunks: S stays in registers (and
//                                in LDS as an operand)
//
// All of it is 32-bit, products included (fp32 MFMA).  No exponent is ever positive: the 16 x 16 blocks on the diagonal of A
// and B weigh every pair of tokens on its own, the blocks under it go through the decay up to the border of the row block,
// e^(G_i - R) e^(R - G_j), whose factors are both at most one.  Tokens behind the end of the portion count as zeros without decay.
#include "dense.h"
#include "dense_kernels.h"

namespace w4a16 {

namespace {

constexpr int kC = 64, kThreads = 256;
constexpr float kLog2E = 1.4426950408889634f;

// Work of one head and chunk, in floats.  The matrices lie in the order in which the scan's waves read them as first operands, a
// kilobyte of neighbouring lanes per load: [16 rows][32 columns][half of 8 columns][lane][4]; u as it is added to a product:
// [16 columns][16 tokens][lane][4 tokens].
struct ChunkLayout {
    int dim, vdim, delta;
    __host__ __device__ size_t q() const { return 0; }                                   // [kC][dim]
    __host__ __device__ size_t k() const { return (size_t)kC * dim; }                    // [dim][kC]
    __host__ __device__ size_t b() const { return k() + (size_t)kC * dim; }              // [kC][kC]
    __host__ __device__ size_t u() const { return b() + kC * kC; }                       // [kC][vdim]
    __host__ __device__ size_t e() const { return u() + (size_t)kC * vdim; }             // [dim]
    __host__ __device__ size_t w() const { return e() + dim; }                           // [kC][dim]
    __host__ __device__ size_t size() const { return w() + (delta ? (size_t)kC * dim : 0); }
};

// Place of elements (row, column .. column + 3) of a matrix with `steps` times 32 columns.
__device__ __forceinline__ int place_of(int row, int col, int steps) {
    return (((row >> 4) * steps + (col >> 5)) * 2 + ((col >> 2) & 1)) * 256 + (((col & 31) >> 3) * 16 + (row & 15)) * 4;
}
// ... and the row and first column of the four elements at place 4 `slot`
__device__ __forceinline__ void at_place(int slot, int steps, int &row, int &col) {
    const int lane = slot & 63, piece = slot >> 6, half = piece & 1, step = (piece >> 1) % steps;
    row = (piece >> 1) / steps * 16 + (lane & 15);
    col = 32 * step + 8 * (lane >> 4) + 4 * half;
}

// zeros of the blocks above the diagonal that the scan reads (columns 16 .. 31 of rows 0 .. 15, 48 .. 63 of rows 32 .. 47)
__device__ __forceinline__ void clear_upper(float *b, int lane) {
    const int row = lane >> 2, c = 4 * (lane & 3);
    const floatx4 zero = floatx4{0.f, 0.f, 0.f, 0.f};
    *reinterpret_cast<floatx4 *>(b + place_of(row, 16 + c, 2)) = zero;
    *reinterpret_cast<floatx4 *>(b + place_of(32 + row, 48 + c, 2)) = zero;
}

// blockIdx.x = chunk, blockIdx.y = head.  One decay per head, u = v.
template <class T, int ND>
__global__ void __launch_bounds__(kThreads) linear_chunk_kernel(const LinearArgs a, const T *q, const T *k, const T *v, float *work) {
    constexpr int D = 64 * ND, P = D + 4;
    __shared__ __attribute__((aligned(16))) float ks[kC][P];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, ql = lane & 15, g = lane >> 4;
    const int h = blockIdx.y, kh = h / (a.heads / a.k_heads), m0 = blockIdx.x * kC, n = a.M - m0 < kC ? a.M - m0 : kC;
    const ChunkLayout lay{D, a.vdim, 0};
    float *out = work + ((size_t)h * gridDim.x + blockIdx.x) * lay.size();
    const float ld = a.log2_decay[h];
    auto power = [&](int e) { return __builtin_amdgcn_exp2f(ld * (float)e); };
    q += (size_t)m0 * a.ld + (size_t)kh * D;
    k += (size_t)m0 * a.ld + (size_t)kh * D;
    v += (size_t)m0 * a.ld + (size_t)h * a.vdim;
    for (int i = tid; i < kC * D / 8; i += kThreads) {
        const int r = i / (D / 8), c = 8 * (i % (D / 8));
        float y[8];
        unpack8(r < n ? load8(k + (size_t)r * a.ld + c) : zero8<T>(), y);
        store8(&ks[r][c], pack8<float>(y));
    }
    for (int i = tid; i < kC * D / 4; i += kThreads) {
        int r, c;
        at_place(i, 2 * ND, r, c);
        float x[4] = {0.f, 0.f, 0.f, 0.f};
        if (r < n) load4(q + (size_t)r * a.ld + c, x);
        const float f = power(r + 1);
        store4(out + lay.q() + 4 * i, x[0] * f, x[1] * f, x[2] * f, x[3] * f);
    }
    for (int i = tid; i < kC * a.vdim / 4; i += kThreads) {
        const int t = 16 * ((i >> 6) & 3) + 4 * ((i & 63) >> 4), c = 16 * (i >> 8) + (i & 15);
        float x[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] = t + e < n ? to_float(v[(size_t)(t + e) * a.ld + c]) : 0.f;
        store4(out + lay.u() + 4 * i, x[0], x[1], x[2], x[3]);
    }
    if (tid < D) out[lay.e() + tid] = power(n);
    // scores: rows of one wave against the blocks up to the diagonal (first operand: k, so that a lane owns one query)
    const int qi = 16 * wave + ql;
    const T *qr = q + (size_t)(qi < n ? qi : n - 1) * a.ld + 8 * g;
    for (int bj = 0; bj <= wave; ++bj) {
        const int kj = 16 * bj + ql;
        const T *kr = k + (size_t)(kj < n ? kj : n - 1) * a.ld + 8 * g;
        floatx4 s = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < 2 * ND; ++t) s = mma32(load8(kr + 32 * t), load8(qr + 32 * t), s);
        float w[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int j = 16 * bj + 4 * g + r;
            w[r] = j <= qi && j < n && qi < n ? s[r] * power(qi - j) : 0.f;
        }
        store4(out + lay.b() + place_of(qi, 16 * bj + 4 * g, 2), w[0], w[1], w[2], w[3]);
    }
    if (wave == 0) clear_upper(out + lay.b(), lane);
    __syncthreads();
    for (int i = tid; i < D * kC / 4; i += kThreads) {
        int r, c;
        at_place(i, 2, c, r);
        float x[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] = r + e < n ? ks[r + e][c] * power(n - 1 - r - e) : 0.f;
        store4(out + lay.k() + 4 * i, x[0], x[1], x[2], x[3]);
    }
}

// The lower triangle of A in 16 x 16 blocks: place of block (i, j), j <= i.
__device__ __forceinline__ constexpr int block_at(int i, int j) { return (i * (i + 1) / 2 + j) * 256; }

// acc + M X with M 16 x 16 (row l % 16, columns 4 (l / 16) .. + 3 in lane l) and X as a product leaves it (rows 4 (l / 16) .. + 3 of
// column l % 16)
__device__ __forceinline__ floatx4 mma16(floatx4 m, floatx4 x, floatx4 acc) {
#pragma unroll
    for (int t = 0; t < 4; ++t) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(m[t], x[t], acc, 0, 0, 0);
    return acc;
}

template <class T, int ND>
struct DeltaLds {
    static constexpr int D = 64 * ND, P = D + 4, KP = D + 16 / (int)sizeof(T);
    float g[kC * P], a[10 * 256], beta[kC], kf[kC], qf[kC];
    T k[kC * KP], q[kC * KP];
};

// blockIdx.x = chunk, blockIdx.y = head.  One decay per channel, the delta rule.
template <class T, int ND>
__global__ void __launch_bounds__(kThreads, sizeof(T) == 2 ? 2 : 1) delta_chunk_kernel(const LinearArgs a, const T *q, const T *k, const T *v, const T *beta,
                                                                                       float *work) {
    using Lds = DeltaLds<T, ND>;
    constexpr int D = Lds::D, P = Lds::P, KP = Lds::KP;
    extern __shared__ __attribute__((aligned(16))) char delta_lds[];
    Lds &s = *reinterpret_cast<Lds *>(delta_lds);
    const int tid = threadIdx.x, lane = tid & 63, ql = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int h = blockIdx.y, kh = h / (a.heads / a.k_heads), m0 = blockIdx.x * kC, n = a.M - m0 < kC ? a.M - m0 : kC;
    const ChunkLayout lay{D, a.vdim, 1};
    float *out = work + ((size_t)h * gridDim.x + blockIdx.x) * lay.size();
    const float ea = -expf(a.a_log[h]) * kLog2E;
    q += (size_t)m0 * a.ld + (size_t)kh * D;
    k += (size_t)m0 * a.ld + (size_t)kh * D;
    v += (size_t)m0 * a.ld + (size_t)h * a.vdim;
    const float *z = a.z + ((size_t)m0 * a.heads + h) * D, *bias = a.dt_bias + (size_t)h * D;
    for (int i = tid; i < kC * D / 8; i += kThreads) {
        const int r = i / (D / 8), c = 8 * (i % (D / 8));
        store8(s.q + r * KP + c, r < n ? load8(q + (size_t)r * a.ld + c) : zero8<T>());
        store8(s.k + r * KP + c, r < n ? load8(k + (size_t)r * a.ld + c) : zero8<T>());
    }
    {   // log2 decays and their sums along the tokens: runs of kC / RUNS tokens, then the runs in front
        constexpr int RUNS = kThreads / D, LEN = kC / RUNS;
        const int c = tid % D, run = tid / D;
        const float b = bias[c];
        float x[LEN], sum = 0.f;
#pragma unroll
        for (int r = 0; r < LEN; ++r) x[r] = run * LEN + r < n ? z[(size_t)(run * LEN + r) * a.heads * D + c] : -1.0e30f;
#pragma unroll
        for (int r = 0; r < LEN; ++r) {
            sum += ea * softplus_f32(x[r] + b);      // (0 behind the end)
            x[r] = sum;
        }
        s.a[tid] = sum;
        if (tid < kC) {
            const float *f = a.factors + (size_t)(m0 + (tid < n ? tid : 0)) * 2 * a.k_heads + kh;
            s.qf[tid] = tid < n ? f[0] : 0.f;
            s.kf[tid] = tid < n ? f[a.k_heads] : 0.f;
            s.beta[tid] = tid < n ? sigmoid_f32(to_float(beta[(size_t)(m0 + tid) * a.ld_beta + h])) : 0.f;
        }
        __syncthreads();
        float front = 0.f;
        for (int i = 0; i < run; ++i) front += s.a[i * D + c];
#pragma unroll
        for (int r = 0; r < LEN; ++r) s.g[(run * LEN + r) * P + c] = front + x[r];
    }
    __syncthreads();

    // Scores of row block bi against the column blocks bj0 .. bj1 - 1 (at most three): -beta A into LDS, B to memory.  Block (bi, bi)
    // goes the same way, through the decay up to its first row, unless that decay is too strong for fp32 within the block.
    auto put = [&](int bi, int bj, floatx4 sa, floatx4 sb) {
        const int i = 16 * bi + ql, j = 16 * bj + 4 * g;
        const floatx4 kf = *reinterpret_cast<const floatx4 *>(s.kf + j);
        const float fa = -s.beta[i] * s.kf[i], fb = s.qf[i];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            sa[r] = bj == bi && 4 * g + r >= ql ? 0.f : sa[r] * (fa * kf[r]);
            sb[r] = bj == bi && 4 * g + r > ql ? 0.f : sb[r] * (fb * kf[r]);
        }
        *reinterpret_cast<floatx4 *>(s.a + block_at(bi, bj) + 16 * ql + 4 * g) = sa;
        *reinterpret_cast<floatx4 *>(out + lay.b() + place_of(i, j, 2)) = sb;
    };
    auto scores = [&](int bi, int bj0, int bj1) {
        const float *ref = s.g + (16 * bi - 1) * P;     // (bi = 0: nothing in front)
        bool by_pairs = false;
        if (bj1 > bi) {
            bool strong = false;
            for (int c = lane; c < D; c += 64) strong = strong || (bi ? ref[c] : 0.f) - s.g[(16 * bi + 15) * P + c] > 100.f;
            by_pairs = __builtin_amdgcn_ballot_w64(strong) != 0;
        }
        const int last = by_pairs ? bi : bj1;
        floatx4 sa[3], sb[3];
#pragma unroll
        for (int t = 0; t < 3; ++t) sa[t] = sb[t] = floatx4{0.f, 0.f, 0.f, 0.f};
        const int i = 16 * bi + ql;
        for (int c = 8 * g; c < D; c += 32) {
            float r[8], x[8], ki[8], qi[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) r[e] = 0.f;
            if (bi) unpack8(load8(ref + c), r);
            unpack8(load8(s.g + i * P + c), x);
            unpack8(load8(s.k + i * KP + c), ki);
            unpack8(load8(s.q + i * KP + c), qi);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float f = __builtin_amdgcn_exp2f(x[e] - r[e]);
                ki[e] *= f;
                qi[e] *= f;
            }
            const Vec8<float> vk = pack8<float>(ki), vq = pack8<float>(qi);
#pragma unroll
            for (int t = 0; t < 3; ++t) {
                if (bj0 + t >= last) continue;
                const int j = 16 * (bj0 + t) + ql;
                float y[8], kj[8];
                unpack8(load8(s.g + j * P + c), y);
                unpack8(load8(s.k + j * KP + c), kj);
#pragma unroll
                for (int e = 0; e < 8; ++e) kj[e] *= __builtin_amdgcn_exp2f(r[e] - y[e]);
                const Vec8<float> vj = pack8<float>(kj);
                sa[t] = mma32(vj, vk, sa[t]);
                sb[t] = mma32(vj, vq, sb[t]);
            }
        }
#pragma unroll
        for (int t = 0; t < 3; ++t)
            if (bj0 + t < last) put(bi, bj0 + t, sa[t], sb[t]);
        if (!by_pairs) return;
        floatx4 da = floatx4{0.f, 0.f, 0.f, 0.f}, db = da;
        const int j0 = 16 * bi + 4 * g;
        for (int c = 0; c < D; c += 4) {
            const floatx4 gi = *reinterpret_cast<const floatx4 *>(s.g + i * P + c);
            float ki[4], qi[4];
            load4(s.k + i * KP + c, ki);
            load4(s.q + i * KP + c, qi);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const floatx4 gj = *reinterpret_cast<const floatx4 *>(s.g + (j0 + r) * P + c);
                float kj[4];
                load4(s.k + (j0 + r) * KP + c, kj);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float t = __builtin_amdgcn_exp2f(fminf(gi[e] - gj[e], 0.f)) * kj[e];
                    da[r] = fmaf(ki[e], t, da[r]);
                    db[r] = fmaf(qi[e], t, db[r]);
                }
            }
        }
        put(bi, bi, da, db);
    };
    if (wave == 0) scores(3, 0, 2);
    else if (wave == 1) scores(3, 2, 4);
    else if (wave == 2) scores(2, 0, 3);
    else {
        scores(1, 0, 2);
        scores(0, 0, 1);
        clear_upper(out + lay.b(), lane);
    }
    __syncthreads();
    {   // the block on the diagonal becomes the inverse of 1 + diag(beta) A there: a lane has one of its columns
        float *blk = s.a + block_at(wave, wave);
        float y[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            y[i] = i == ql ? 1.f : 0.f;
#pragma unroll
            for (int j = 0; j < i; j += 4) {
                const floatx4 l = *reinterpret_cast<const floatx4 *>(blk + 16 * i + j);
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (j + e < i) y[i] = fmaf(l[e], y[j + e], y[i]);
            }
        }
        if (g == 0) {
#pragma unroll
            for (int i = 0; i < 16; ++i) blk[16 * i + ql] = y[i];
        }
    }
    __syncthreads();
    // (1 + diag(beta) A) X = right-hand side by blocks of 16 tokens, 16 columns at a time: k e^G (W), then v (U0)
    floatx4 m[10];
#pragma unroll
    for (int i = 0; i < 10; ++i) m[i] = *reinterpret_cast<const floatx4 *>(s.a + 256 * i + 16 * ql + 4 * g);
    auto solve = [&](floatx4 (&x)[4]) {
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            floatx4 acc = x[b];
#pragma unroll
            for (int j = 0; j < b; ++j) acc = mma16(m[block_at(b, j) / 256], x[j], acc);
            x[b] = mma16(m[block_at(b, b) / 256], acc, floatx4{0.f, 0.f, 0.f, 0.f});
        }
    };
    floatx4 w[ND][4];
#pragma unroll
    for (int ct = 0; ct < ND; ++ct) {
        const int c = 16 * (wave + 4 * ct) + ql;
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            const int i = 16 * b + 4 * g;
            const floatx4 be = *reinterpret_cast<const floatx4 *>(s.beta + i), kf = *reinterpret_cast<const floatx4 *>(s.kf + i);
#pragma unroll
            for (int r = 0; r < 4; ++r) w[ct][b][r] = be[r] * kf[r] * to_float(s.k[(i + r) * KP + c]) * __builtin_amdgcn_exp2f(s.g[(i + r) * P + c]);
        }
        solve(w[ct]);
    }
    for (int vt = wave; vt < a.vdim / 16; vt += 4) {
        floatx4 x[4];
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            const int i = 16 * b + 4 * g;
            const floatx4 be = *reinterpret_cast<const floatx4 *>(s.beta + i);
#pragma unroll
            for (int r = 0; r < 4; ++r) x[b][r] = be[r] * to_float(v[(size_t)(i + r < n ? i + r : n - 1) * a.ld + 16 * vt + ql]);   // (beta is 0 from n on)
        }
        solve(x);
#pragma unroll
        for (int b = 0; b < 4; ++b) *reinterpret_cast<floatx4 *>(out + lay.u() + ((vt * 4 + b) * 64 + lane) * 4) = x[b];
    }
    const float *end = s.g + (kC - 1) * P;
    for (int i = tid; i < kC * D / 4; i += kThreads) {
        int r, c;
        at_place(i, 2 * ND, r, c);
        const floatx4 x = *reinterpret_cast<const floatx4 *>(s.g + r * P + c);
        const float f = s.qf[r];
        float y[4];
        load4(s.q + r * KP + c, y);
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] *= f * __builtin_amdgcn_exp2f(x[e]);
        store4(out + lay.q() + 4 * i, y[0], y[1], y[2], y[3]);
    }
    for (int i = tid; i < kC * D / 4; i += kThreads) {
        int r, c;
        at_place(i, 2, c, r);
        float y[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] = s.kf[r + e] * to_float(s.k[(r + e) * KP + c]) * __builtin_amdgcn_exp2f(end[c] - s.g[(r + e) * P + c]);
        store4(out + lay.k() + 4 * i, y[0], y[1], y[2], y[3]);
    }
    if (tid < D) out[lay.e() + tid] = __builtin_amdgcn_exp2f(end[tid]);
    __syncthreads();   // the decays make room for W on its way into another order
#pragma unroll
    for (int ct = 0; ct < ND; ++ct)
#pragma unroll
        for (int b = 0; b < 4; ++b)
#pragma unroll
            for (int r = 0; r < 4; ++r) s.g[(16 * b + 4 * g + r) * P + 16 * (wave + 4 * ct) + ql] = w[ct][b][r];
    __syncthreads();
    for (int i = tid; i < kC * D / 4; i += kThreads) {
        int r, c;
        at_place(i, 2 * ND, r, c);
        *reinterpret_cast<floatx4 *>(out + lay.w() + 4 * i) = *reinterpret_cast<const floatx4 *>(s.g + r * P + c);
    }
}

// A workgroup: 16 value columns of a head; those of one head run on one XCD, whose L2 the head's operands go through once.  Four waves
// bring the state forward (16 tokens each in the product with W, the key channels 16 (wave + 4 c) .. + 15 of S each), four make the
// outputs (16 tokens each); a SIMD has one of either, which fill each other's waits.  S and U go through LDS, two buffers each.
// A wave requests the operands of the next chunk as soon as it has multiplied those of this one, products with S while those with U
// are made and the other way round.  (Behind the last chunk that one is fetched again rather than nothing, so that the number of loads
// in flight is known at every wait.)
template <int ND, bool DELTA>
__global__ void __launch_bounds__(2 * kThreads, 1) chunk_scan_kernel(const LinearArgs a, const float *work, int chunks, bool first, float *o) {
    constexpr int D = 64 * ND, KS = 2 * ND;
    __shared__ __attribute__((aligned(16))) float ss[2][16][D + 4], us[2][16][kC + 4];
    const int tid = threadIdx.x, lane = tid & 63, ql = lane & 15, g = lane >> 4;
    const int wave8 = __builtin_amdgcn_readfirstlane(tid >> 6), wave = wave8 & 3;
    const int tiles = a.vdim / 16, xcd = blockIdx.x & 7, at = blockIdx.x >> 3;
    const int h = 8 * (at / tiles) + xcd, v0 = 16 * (at % tiles), tok = 16 * wave;
    if (h >= a.heads) return;
    const ChunkLayout lay{D, a.vdim, DELTA};
    work += (size_t)h * chunks * lay.size();
    auto operand = [&](const float *m, int piece) {
        const float *x = m + piece * 512 + lane * 4;
        return Vec8<float>{*reinterpret_cast<const floatx4 *>(x), *reinterpret_cast<const floatx4 *>(x + 256)};
    };
    const floatx4 zero = floatx4{0.f, 0.f, 0.f, 0.f};
    // m S (two chains), and the operands from LDS in registers before the first product: the compiler would fetch them two by two
    auto times_state = [&](const Vec8<float> (&m)[KS], const float (*rows)[D + 4], floatx4 &x, floatx4 &y) {
        Vec8<float> sv[KS];
#pragma unroll
        for (int t = 0; t < KS; ++t) sv[t] = load8(&rows[ql][32 * t + 8 * g]);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int t = 0; t < KS; t += 2) {
            x = mma32(m[t], sv[t], x);
            y = mma32(m[t + 1], sv[t + 1], y);
        }
    };

    if (wave8 < 4) {
        float *st = a.state + ((size_t)h * a.vdim + v0 + ql) * D + 4 * g;
        const bool from_zero = first && (a.pos_dev ? a.pos_dev[0] : a.pos) == 0;
        floatx4 s[ND];
#pragma unroll
        for (int c = 0; c < ND; ++c) {
            s[c] = from_zero ? zero : *reinterpret_cast<const floatx4 *>(st + 16 * (wave + 4 * c));
            *reinterpret_cast<floatx4 *>(&ss[0][ql][16 * (wave + 4 * c) + 4 * g]) = s[c];
        }
        Vec8<float> w[KS], k[ND][2];   // (w: the delta rule only)
        floatx4 u, e[ND];
        auto fetch_w = [&](const float *p) {
            if constexpr (DELTA) {
#pragma unroll
                for (int t = 0; t < KS; ++t) w[t] = operand(p + lay.w(), wave * KS + t);
            }
            u = *reinterpret_cast<const floatx4 *>(p + lay.u() + ((v0 / 16 * 4 + wave) * 64 + lane) * 4);
#pragma unroll
            for (int c = 0; c < ND; ++c) e[c] = *reinterpret_cast<const floatx4 *>(p + lay.e() + 16 * (wave + 4 * c) + 4 * g);
        };
        auto fetch_k = [&](const float *p) {
#pragma unroll
            for (int c = 0; c < ND; ++c)
#pragma unroll
                for (int t = 0; t < 2; ++t) k[c][t] = operand(p + lay.k(), (wave + 4 * c) * 2 + t);
        };
        fetch_w(work);
        fetch_k(work);
        if constexpr (!DELTA) *reinterpret_cast<floatx4 *>(&us[0][ql][tok + 4 * g]) = u;
        __syncthreads();
        for (int chunk = 0; chunk < chunks; ++chunk) {
            const int b = chunk & 1;
            work += chunk + 1 < chunks ? lay.size() : 0;
#pragma unroll
            for (int c = 0; c < ND; ++c) s[c] *= e[c];
            if constexpr (DELTA) {
                floatx4 x = zero, y = zero;
                times_state(w, ss[b], x, y);
                *reinterpret_cast<floatx4 *>(&us[b][ql][tok + 4 * g]) = u - (x + y);
                fetch_w(work);
                __syncthreads();   // U is there
            } else {
                fetch_w(work);
            }
            const Vec8<float> ua = load8(&us[b][ql][8 * g]), ub = load8(&us[b][ql][32 + 8 * g]);
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int c = 0; c < ND; ++c) s[c] = mma32(k[c][0], ua, s[c]);
#pragma unroll
            for (int c = 0; c < ND; ++c) {
                s[c] = mma32(k[c][1], ub, s[c]);
                *reinterpret_cast<floatx4 *>(&ss[b ^ 1][ql][16 * (wave + 4 * c) + 4 * g]) = s[c];
            }
            fetch_k(work);
            if constexpr (!DELTA) *reinterpret_cast<floatx4 *>(&us[b ^ 1][ql][tok + 4 * g]) = u;
            __syncthreads();       // the next S (and, without the delta rule, U) is there, this one has been read
        }
#pragma unroll
        for (int c = 0; c < ND; ++c) *reinterpret_cast<floatx4 *>(st + 16 * (wave + 4 * c)) = s[c];
    } else {
        Vec8<float> q[KS], m[2];
        auto fetch_q = [&](const float *p) {
#pragma unroll
            for (int t = 0; t < KS; ++t) q[t] = operand(p + lay.q(), wave * KS + t);
        };
        auto fetch_b = [&](const float *p) {
#pragma unroll
            for (int t = 0; t < 2; ++t) m[t] = operand(p + lay.b(), wave * 2 + t);   // (the first two waves use one)
        };
        fetch_q(work);
        fetch_b(work);
        o += (size_t)(tok + 4 * g) * a.heads * a.vdim + (size_t)h * a.vdim + v0 + ql;
        __syncthreads();
        for (int chunk = 0; chunk < chunks; ++chunk) {
            const int b = chunk & 1;
            work += chunk + 1 < chunks ? lay.size() : 0;
            floatx4 x = zero, y = zero;
            times_state(q, ss[b], x, y);
            fetch_q(work);
            if constexpr (DELTA) __syncthreads();
            const Vec8<float> ua = load8(&us[b][ql][8 * g]), ub = load8(&us[b][ql][32 + 8 * g]);
            x = mma32(m[0], ua, x);
            if (wave >= 2) y = mma32(m[1], ub, y);
            fetch_b(work);
            x += y;
            const int row = chunk * kC + tok + 4 * g;
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (row + r < a.M) o[(size_t)(chunk * kC + r) * a.heads * a.vdim] = x[r];
            __syncthreads();
        }
    }
}

// Chunks that are worked on at once: their operands stay within reach of the last-level cache.
int segment_chunks(const LinearArgs &a) {
    const ChunkLayout lay{a.dim, a.vdim, a.z != nullptr};
    const size_t per = lay.size() * sizeof(float) * a.heads;
    const int all = (a.M + kC - 1) / kC, fit = (int)((size_t)160 * 1024 * 1024 / per);
    return all < fit ? all : fit < 8 ? (all < 8 ? all : 8) : fit;
}

template <class T, int ND>
hipError_t chunks(LinearArgs a, float *work, float *o, hipStream_t stream) {
    const int seg = segment_chunks(a), M = a.M;
    const T *qkv = static_cast<const T *>(a.qkv), *beta = static_cast<const T *>(a.beta);
    constexpr size_t lds = sizeof(DeltaLds<T, ND>);
    if (a.z && lds > 48 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(&delta_chunk_kernel<T, ND>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    for (int m0 = 0; m0 < M; m0 += seg * kC) {
        a.M = M - m0 < seg * kC ? M - m0 : seg * kC;
        const int n = (a.M + kC - 1) / kC;
        const dim3 grid(n, a.heads), scan(8 * ((a.heads + 7) / 8) * (a.vdim / 16));
        const T *q = qkv + (size_t)m0 * a.ld + a.q_off, *k = qkv + (size_t)m0 * a.ld + a.k_off, *v = qkv + (size_t)m0 * a.ld + a.v_off;
        float *om = o + (size_t)m0 * a.heads * a.vdim;
        if (a.z) {
            LinearArgs b = a;
            b.z += (size_t)m0 * a.heads * a.dim;
            b.factors += (size_t)m0 * 2 * a.k_heads;
            hipLaunchKernelGGL((delta_chunk_kernel<T, ND>), grid, dim3(kThreads), lds, stream, b, q, k, v, beta + (size_t)m0 * a.ld_beta, work);
            hipLaunchKernelGGL((chunk_scan_kernel<ND, true>), scan, dim3(2 * kThreads), 0, stream, a, work, n, m0 == 0, om);
        } else {
            hipLaunchKernelGGL((linear_chunk_kernel<T, ND>), grid, dim3(kThreads), 0, stream, a, q, k, v, work);
            hipLaunchKernelGGL((chunk_scan_kernel<ND, false>), scan, dim3(2 * kThreads), 0, stream, a, work, n, m0 == 0, om);
        }
        const hipError_t e = hipGetLastError();
        if (e != hipSuccess) return e;
    }
    return hipSuccess;
}

}  // namespace

bool linear_chunks_supported(const LinearArgs &a) { return a.dim <= 128; }

size_t linear_chunk_bytes(const LinearArgs &a) {
    const ChunkLayout lay{a.dim, a.vdim, a.z != nullptr};
    return lay.size() * sizeof(float) * a.heads * segment_chunks(a);
}

hipError_t launch_linear_chunks(int dtype, const LinearArgs &a, void *work, float *o, hipStream_t stream) {
    float *w = static_cast<float *>(work);
    if (dtype == kF32) return a.dim == 64 ? chunks<float, 1>(a, w, o, stream) : chunks<float, 2>(a, w, o, stream);
    return a.dim == 64 ? chunks<bf16, 1>(a, w, o, stream) : chunks<bf16, 2>(a, w, o, stream);
}

}  // namespace w4a16
