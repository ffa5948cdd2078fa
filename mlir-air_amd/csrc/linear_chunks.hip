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
//                                in LDS as an operand), the next chunk's operands travel while one is multiplied
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

// Work of one head and chunk, in floats.
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

// zeros of the blocks above the diagonal that the scan reads (columns 16 .. 31 of rows 0 .. 15, 48 .. 63 of rows 32 .. 47)
__device__ __forceinline__ void clear_upper(float *b, int lane) {
    const int r = lane >> 2, c = 4 * (lane & 3);
    const floatx4 zero = floatx4{0.f, 0.f, 0.f, 0.f};
    *reinterpret_cast<floatx4 *>(b + r * kC + 16 + c) = zero;
    *reinterpret_cast<floatx4 *>(b + (32 + r) * kC + 48 + c) = zero;
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
    for (int i = tid; i < kC * D / 4; i += kThreads) {
        const int r = i / (D / 4), c = 4 * (i % (D / 4));
        float x[4] = {0.f, 0.f, 0.f, 0.f}, y[4] = {0.f, 0.f, 0.f, 0.f};
        if (r < n) {
            load4(q + (size_t)r * a.ld + c, x);
            load4(k + (size_t)r * a.ld + c, y);
        }
        const float f = power(r + 1);
        store4(out + lay.q() + r * D + c, x[0] * f, x[1] * f, x[2] * f, x[3] * f);
        store4(&ks[r][c], y[0], y[1], y[2], y[3]);
    }
    for (int i = tid; i < kC * a.vdim / 4; i += kThreads) {
        const int r = i / (a.vdim / 4), c = 4 * (i % (a.vdim / 4));
        float x[4] = {0.f, 0.f, 0.f, 0.f};
        if (r < n) load4(v + (size_t)r * a.ld + c, x);
        store4(out + lay.u() + (size_t)r * a.vdim + c, x[0], x[1], x[2], x[3]);
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
        store4(out + lay.b() + qi * kC + 16 * bj + 4 * g, w[0], w[1], w[2], w[3]);
    }
    if (wave == 0) clear_upper(out + lay.b(), lane);
    __syncthreads();
    for (int i = tid; i < D * kC; i += kThreads) {
        const int c = i / kC, r = i % kC;
        out[lay.k() + i] = r < n ? ks[r][c] * power(n - 1 - r) : 0.f;
    }
}

// blockIdx.x = chunk, blockIdx.y = head.  One decay per channel, the delta rule.
template <class T, int ND>
__global__ void __launch_bounds__(kThreads) delta_chunk_kernel(const LinearArgs a, const T *q, const T *k, const T *v, const T *beta, float *work) {
    constexpr int D = 64 * ND, P = D + 4, LP = kC + 4;
    extern __shared__ __attribute__((aligned(16))) float delta_lds[];
    float *gs = delta_lds, *ks = gs + kC * P, *qs = ks + kC * P, *ls = qs + kC * P, *bs = ls + kC * LP;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, ql = lane & 15, g = lane >> 4;
    const int h = blockIdx.y, kh = h / (a.heads / a.k_heads), m0 = blockIdx.x * kC, n = a.M - m0 < kC ? a.M - m0 : kC;
    const ChunkLayout lay{D, a.vdim, 1};
    float *out = work + ((size_t)h * gridDim.x + blockIdx.x) * lay.size();
    const float ea = -expf(a.a_log[h]) * kLog2E;
    q += (size_t)m0 * a.ld + (size_t)kh * D;
    k += (size_t)m0 * a.ld + (size_t)kh * D;
    v += (size_t)m0 * a.ld + (size_t)h * a.vdim;
    const float *z = a.z + ((size_t)m0 * a.heads + h) * D, *bias = a.dt_bias + (size_t)h * D;
    for (int i = tid; i < kC * D / 4; i += kThreads) {
        const int r = i / (D / 4), c = 4 * (i % (D / 4));
        float x[4] = {0.f, 0.f, 0.f, 0.f}, y[4] = {0.f, 0.f, 0.f, 0.f}, l[4] = {0.f, 0.f, 0.f, 0.f};
        if (r < n) {
            load4(q + (size_t)r * a.ld + c, x);
            load4(k + (size_t)r * a.ld + c, y);
            float b[4];
            load4(z + (size_t)r * a.heads * D + c, l);
            load4(bias + c, b);
            const float *f = a.factors + (size_t)(m0 + r) * 2 * a.k_heads + kh;
            const float qf = f[0], kf = f[a.k_heads];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                x[e] *= qf;
                y[e] *= kf;
                l[e] = ea * softplus_f32(l[e] + b[e]);
            }
        }
        store4(qs + r * P + c, x[0], x[1], x[2], x[3]);
        store4(ks + r * P + c, y[0], y[1], y[2], y[3]);
        store4(gs + r * P + c, l[0], l[1], l[2], l[3]);
    }
    if (tid < kC) bs[tid] = tid < n ? sigmoid_f32(to_float(beta[(size_t)(m0 + tid) * a.ld_beta + h])) : 0.f;
    __syncthreads();
    {   // sums along the tokens: runs of kC / RUNS tokens, then the runs in front
        constexpr int RUNS = kThreads / D, LEN = kC / RUNS;
        const int c = tid % D, run = tid / D;
        float s = 0.f;
        for (int r = run * LEN; r < (run + 1) * LEN; ++r) {
            s += gs[r * P + c];
            gs[r * P + c] = s;
        }
        __syncthreads();
        float front = 0.f;
        for (int i = 0; i < run; ++i) front += gs[((i + 1) * LEN - 1) * P + c];
        __syncthreads();
        for (int r = run * LEN; r < (run + 1) * LEN; ++r) gs[r * P + c] += front;
    }
    __syncthreads();
    // a lane's scores: row i against columns j0 .. j0 + 3
    auto put = [&](int i, int j0, floatx4 sa, floatx4 sb) {
        const float bi = bs[i];
        store4(ls + i * LP + j0, sa[0] * bi, sa[1] * bi, sa[2] * bi, sa[3] * bi);
        store4(out + lay.b() + i * kC + j0, sb[0], sb[1], sb[2], sb[3]);
    };
    {
        const int i = 16 * wave + ql, j0 = 16 * wave + 4 * g;
        floatx4 sa = floatx4{0.f, 0.f, 0.f, 0.f}, sb = sa;
        for (int c = 0; c < D; c += 4) {
            const floatx4 gi = *reinterpret_cast<const floatx4 *>(gs + i * P + c), ki = *reinterpret_cast<const floatx4 *>(ks + i * P + c),
                          qi = *reinterpret_cast<const floatx4 *>(qs + i * P + c);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const floatx4 gj = *reinterpret_cast<const floatx4 *>(gs + (j0 + r) * P + c), kj = *reinterpret_cast<const floatx4 *>(ks + (j0 + r) * P + c);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float t = __builtin_amdgcn_exp2f(fminf(gi[e] - gj[e], 0.f)) * kj[e];
                    sa[r] = fmaf(ki[e], t, sa[r]);
                    sb[r] = fmaf(qi[e], t, sb[r]);
                }
            }
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            if (j0 + r >= i) sa[r] = 0.f;
            if (j0 + r > i) sb[r] = 0.f;
        }
        put(i, j0, sa, sb);
    }
    for (int b = wave; b < 6; b += 4) {
        const int bi = b < 3 ? 3 : b < 5 ? 2 : 1, bj = b < 3 ? b : b < 5 ? b - 3 : 0;
        const int i = 16 * bi + ql, j = 16 * bj + ql;
        floatx4 sa = floatx4{0.f, 0.f, 0.f, 0.f}, sb = sa;
        for (int c = 8 * g; c < D; c += 32) {
            float ref[8], gi[8], gj[8], ki[8], qi[8], kj[8];
            unpack8(load8(gs + (16 * bi - 1) * P + c), ref);
            unpack8(load8(gs + i * P + c), gi);
            unpack8(load8(gs + j * P + c), gj);
            unpack8(load8(ks + i * P + c), ki);
            unpack8(load8(qs + i * P + c), qi);
            unpack8(load8(ks + j * P + c), kj);
            Vec8<float> vk, vq, vj;
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float fi = __builtin_amdgcn_exp2f(gi[e] - ref[e]), fj = __builtin_amdgcn_exp2f(ref[e] - gj[e]) * kj[e];
                if (e < 4) {
                    vk.lo[e] = ki[e] * fi;
                    vq.lo[e] = qi[e] * fi;
                    vj.lo[e] = fj;
                } else {
                    vk.hi[e - 4] = ki[e] * fi;
                    vq.hi[e - 4] = qi[e] * fi;
                    vj.hi[e - 4] = fj;
                }
            }
            sa = mma32(vj, vk, sa);
            sb = mma32(vj, vq, sb);
        }
        put(i, 16 * bj + 4 * g, sa, sb);
    }
    if (wave == 3) clear_upper(out + lay.b(), lane);
    __syncthreads();
    // (1 + diag(beta) A) x = right-hand side, one column per thread: k e^G (W), then v (U0)
    for (int c = tid; c < D + a.vdim; c += kThreads) {
        float x[kC];
        if (c < D) {
#pragma unroll
            for (int i = 0; i < kC; ++i) x[i] = bs[i] * ks[i * P + c] * __builtin_amdgcn_exp2f(gs[i * P + c]);
        } else {
            const T *row = v + c - D;
#pragma unroll
            for (int i = 0; i < kC; ++i) {
                x[i] = bs[i] * to_float(*row);   // (beta is 0 from n on)
                row += i + 1 < n ? a.ld : 0;
            }
        }
#pragma unroll
        for (int i = 1; i < kC; ++i) {
            asm volatile("" ::: "memory");   // the rows of A are read as they are needed, not all at once
#pragma unroll
            for (int j = 0; j < i; j += 4) {
                const floatx4 l = *reinterpret_cast<const floatx4 *>(ls + i * LP + j);
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (j + e < i) x[i] = fmaf(-l[e], x[j + e], x[i]);
            }
        }
        float *dst = c < D ? out + lay.w() + c : out + lay.u() + c - D;
        const int ld = c < D ? D : a.vdim;
#pragma unroll
        for (int i = 0; i < kC; ++i, dst += ld) *dst = x[i];
    }
    const float *last = gs + (kC - 1) * P;
    for (int i = tid; i < kC * D; i += kThreads) {
        const int r = i / D, c = i % D;
        out[lay.q() + i] = qs[r * P + c] * __builtin_amdgcn_exp2f(gs[r * P + c]);
    }
    for (int i = tid; i < kC * D; i += kThreads) {
        const int c = i / kC, r = i % kC;
        out[lay.k() + i] = ks[r * P + c] * __builtin_amdgcn_exp2f(last[c] - gs[r * P + c]);
    }
    if (tid < D) out[lay.e() + tid] = __builtin_amdgcn_exp2f(last[tid]);
}

// blockIdx.x = 16 value columns, blockIdx.y = head.  A wave owns 16 tokens of a chunk in the products with S and B, and the key
// channels 16 (wave + 4 c) .. + 15 of S.
template <int ND, bool DELTA>
__global__ void __launch_bounds__(kThreads, 1) chunk_scan_kernel(const LinearArgs a, const float *work, int chunks, bool first, float *o) {
    constexpr int D = 64 * ND, KS = 2 * ND;
    __shared__ __attribute__((aligned(16))) float ss[16][D + 4], us[16][kC + 4];
    const int tid = threadIdx.x, lane = tid & 63, ql = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int h = blockIdx.y, v0 = blockIdx.x * 16, tok = 16 * wave;
    const ChunkLayout lay{D, a.vdim, DELTA};
    work += (size_t)h * chunks * lay.size();
    float *st = a.state + ((size_t)h * a.vdim + v0 + ql) * D + 4 * g;
    const bool from_zero = first && (a.pos_dev ? a.pos_dev[0] : a.pos) == 0;
    floatx4 s[ND];
#pragma unroll
    for (int c = 0; c < ND; ++c) {
        s[c] = from_zero ? floatx4{0.f, 0.f, 0.f, 0.f} : *reinterpret_cast<const floatx4 *>(st + 16 * (wave + 4 * c));
        *reinterpret_cast<floatx4 *>(&ss[ql][16 * (wave + 4 * c) + 4 * g]) = s[c];
    }
    struct Operands {
        Vec8<float> w[DELTA ? KS : 1], q[KS], k[ND][2], b[2];
        floatx4 u, e[ND];
    };
    auto fetch = [&](int chunk, Operands &x) {
        const float *p = work + (size_t)chunk * lay.size();
#pragma unroll
        for (int t = 0; t < KS; ++t) {
            if constexpr (DELTA) x.w[t] = load8(p + lay.w() + (tok + ql) * D + 32 * t + 8 * g);
            x.q[t] = load8(p + lay.q() + (tok + ql) * D + 32 * t + 8 * g);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) x.u[r] = p[lay.u() + (size_t)(tok + 4 * g + r) * a.vdim + v0 + ql];
#pragma unroll
        for (int t = 0; t < 2; ++t)
            if (t == 0 || wave >= 2) x.b[t] = load8(p + lay.b() + (tok + ql) * kC + 32 * t + 8 * g);
#pragma unroll
        for (int c = 0; c < ND; ++c) {
            const int d = 16 * (wave + 4 * c);
#pragma unroll
            for (int t = 0; t < 2; ++t) x.k[c][t] = load8(p + lay.k() + (d + ql) * kC + 32 * t + 8 * g);
            x.e[c] = *reinterpret_cast<const floatx4 *>(p + lay.e() + d + 4 * g);
        }
    };
    auto run = [&](int chunk, const Operands &x) {
        floatx4 acc = floatx4{0.f, 0.f, 0.f, 0.f}, out = acc;
#pragma unroll
        for (int t = 0; t < KS; ++t) {
            const Vec8<float> sv = load8(&ss[ql][32 * t + 8 * g]);
            if constexpr (DELTA) acc = mma32(x.w[t], sv, acc);
            out = mma32(x.q[t], sv, out);
        }
        const floatx4 u = x.u - acc;
        *reinterpret_cast<floatx4 *>(&us[ql][tok + 4 * g]) = u;
        __syncthreads();   // U is there; S has been read by every wave
        const Vec8<float> u0 = load8(&us[ql][8 * g]), u1 = load8(&us[ql][32 + 8 * g]);
#pragma unroll
        for (int c = 0; c < ND; ++c) {
            s[c] = mma32(x.k[c][0], u0, s[c] * x.e[c]);
            s[c] = mma32(x.k[c][1], u1, s[c]);
            *reinterpret_cast<floatx4 *>(&ss[ql][16 * (wave + 4 * c) + 4 * g]) = s[c];
        }
        out = mma32(x.b[0], u0, out);
        if (wave >= 2) out = mma32(x.b[1], u1, out);
        const int m = chunk * kC + tok + 4 * g;
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (m + r < a.M) o[(size_t)(m + r) * a.heads * a.vdim + (size_t)h * a.vdim + v0 + ql] = out[r];
        __syncthreads();
    };
    Operands x, y;
    fetch(0, x);
    __syncthreads();
    for (int c = 0; c < chunks; c += 2) {
        if (c + 1 < chunks) fetch(c + 1, y);
        run(c, x);
        if (c + 1 >= chunks) break;
        if (c + 2 < chunks) fetch(c + 2, x);
        run(c + 1, y);
    }
#pragma unroll
    for (int c = 0; c < ND; ++c) *reinterpret_cast<floatx4 *>(st + 16 * (wave + 4 * c)) = s[c];
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
    constexpr int D = 64 * ND;
    constexpr size_t lds = (size_t)(3 * kC * (D + 4) + kC * (kC + 4) + kC) * sizeof(float);
    if (a.z && lds > 48 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(&delta_chunk_kernel<T, ND>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    for (int m0 = 0; m0 < M; m0 += seg * kC) {
        a.M = M - m0 < seg * kC ? M - m0 : seg * kC;
        const int n = (a.M + kC - 1) / kC;
        const dim3 grid(n, a.heads), scan(a.vdim / 16, a.heads);
        const T *q = qkv + (size_t)m0 * a.ld + a.q_off, *k = qkv + (size_t)m0 * a.ld + a.k_off, *v = qkv + (size_t)m0 * a.ld + a.v_off;
        float *om = o + (size_t)m0 * a.heads * a.vdim;
        if (a.z) {
            LinearArgs b = a;
            b.z += (size_t)m0 * a.heads * a.dim;
            b.factors += (size_t)m0 * 2 * a.k_heads;
            hipLaunchKernelGGL((delta_chunk_kernel<T, ND>), grid, dim3(kThreads), lds, stream, b, q, k, v, beta + (size_t)m0 * a.ld_beta, work);
            hipLaunchKernelGGL((chunk_scan_kernel<ND, true>), scan, dim3(kThreads), 0, stream, a, work, n, m0 == 0, om);
        } else {
            hipLaunchKernelGGL((linear_chunk_kernel<T, ND>), grid, dim3(kThreads), 0, stream, a, q, k, v, work);
            hipLaunchKernelGGL((chunk_scan_kernel<ND, false>), scan, dim3(kThreads), 0, stream, a, work, n, m0 == 0, om);
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
