// Latent attention over the cache for gfx950: the cache holds, per token, one normed latent (rank) and one rotated key part
// (rot) shared by all heads; keys and values of a head are linear in the latent.
//
//   latent_prepare   rotates the queries of many rows in place and appends their cache rows (long portions; keys and values
//                    are then expanded per head and latent_prefill.hip attends)
//   latent_absorb    appends the cache rows and moves the key projection to the query side: qa = W_uk^T q_unrotated per head,
//                    followed by the rotated part, so that a score is one product of length rank + rot with a cache row
//   latent_decode    attention of all rows and heads over the cached rows: HBM-bound on the cache, which is read once per
//                    16 (row, head) pairs; both products on MFMA, keys split over workgroups.  The kernel is the one of every
//                    cache whose rows hold a part that is scored and a part that is summed: for latents they overlap, for
//                    grouped keys and values (head_attention.hip) they lie side by side, in one matrix per key / value head,
//                    and the keys may be limited to a window and kept in a ring of rows
//   latent_combine   merges the splits with the sink, applies the value projection of the head to the merged latent and the
//                    output gate
//
// Positions count from `pos`, which may lie on the device (a captured decode step advances it there).
#include "dense.h"
#include "dense_kernels.h"

namespace w4a16 {

namespace {

constexpr int kLatThreads = 256;

template <class T>
struct LatentArgs {
    LatentShape s;
    const T *proj;
    long ld;
    int kv_off, gate_off;
    const float *lut, *kv_norm;
    float eps;
    T *cache;
    int M;
    const int32_t *pos_dev;
    int pos;
};

template <class T>
__device__ __forceinline__ int first_position(const LatentArgs<T> &p) { return p.pos_dev ? p.pos_dev[0] : p.pos; }

// neighbouring pairs rotated: (u, v) -> (u cos - v sin, v cos + u sin)
template <class T>
__device__ __forceinline__ void rotate_pair(const T *src, T *dst, const float *lut) {
    const float u = to_float(src[0]), v = to_float(src[1]), c = lut[0], s = lut[1];
    dst[0] = from_float<T>(u * c - v * s);
    dst[1] = from_float<T>(v * c + u * s);
}

// The cache row of token m: by one workgroup.  Padding columns of the projections are zeros and stay zeros.
template <class T>
__device__ __forceinline__ void append_row(const LatentArgs<T> &p, int m, int position, float *red) {
    const T *src = p.proj + (size_t)m * p.ld + p.kv_off;
    T *dst = p.cache + (size_t)position * (p.s.rank + p.s.rot);
    float ss = 0.f;
    for (int i = threadIdx.x; i < p.s.rank; i += kLatThreads) {
        const float v = to_float(src[i]);
        ss = fmaf(v, v, ss);
    }
    ss = wave_reduce<false>(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    const float rstd = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)p.s.true_rank + p.eps);
    for (int i = threadIdx.x; i < p.s.rank; i += kLatThreads) dst[i] = from_float<T>(to_float(src[i]) * rstd * p.kv_norm[i]);
    for (int i = threadIdx.x; i < p.s.rot / 2; i += kLatThreads) {
        T *d = dst + p.s.rank + 2 * i;
        if (i < p.s.rot_pairs) rotate_pair(src + p.s.rank + 2 * i, d, p.lut + ((size_t)position * p.s.rot_pairs + i) * 2);
        else d[0] = d[1] = from_float<T>(0.f);
    }
}

// one workgroup per token
template <class T>
__global__ void __launch_bounds__(kLatThreads) latent_prepare_kernel(const LatentArgs<T> p) {
    __shared__ float red[4];
    const int m = blockIdx.x, position = first_position(p) + m;
    const int n = p.s.heads * p.s.rot_pairs, qd = p.s.dim + p.s.rot;
    T *q = const_cast<T *>(p.proj) + (size_t)m * p.ld;
    for (int i = threadIdx.x; i < n; i += kLatThreads) {
        const int h = i / p.s.rot_pairs, j = i % p.s.rot_pairs;
        T *v = q + h * qd + p.s.dim + 2 * j;
        rotate_pair(v, v, p.lut + ((size_t)position * p.s.rot_pairs + j) * 2);
    }
    if (p.kv_off >= 0) append_row(p, m, position, red);
}

// blockIdx.y = token; blockIdx.x = head * blocks of 128 latent columns, then (with a latent of its own) the cache row
template <class T>
__global__ void __launch_bounds__(kLatThreads) latent_absorb_kernel(const LatentArgs<T> p, const T *w_uk, T *qa, int rank_blocks) {
    __shared__ float part[16][128 + 4];
    __shared__ float red[4];
    __shared__ float qs[1024];
    const int m = blockIdx.y, position = first_position(p) + m, tid = threadIdx.x;
    if ((int)blockIdx.x == p.s.heads * rank_blocks) {
        append_row(p, m, position, red);
        return;
    }
    const int h = blockIdx.x / rank_blocks, r0 = (blockIdx.x % rank_blocks) * 128;
    const int qd = p.s.dim + p.s.rot, lq = p.s.rank + p.s.rot;
    const T *q = p.proj + (size_t)m * p.ld + h * qd;
    T *out = qa + ((size_t)m * p.s.heads + h) * lq;
    const int col = r0 + 8 * (tid & 15), dg = tid >> 4;
    float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    for (int i = tid; i < p.s.dim; i += kLatThreads) qs[i] = to_float(q[i]);
    __syncthreads();
    if (col < p.s.rank) {
        const T *w = w_uk + ((size_t)h * p.s.dim + dg) * p.s.rank + col;
        for (int d = dg; d < p.s.dim; d += 64) {       // dim is a multiple of 32: two or four rows at a time
            Vec8<T> v[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) v[j] = d + 16 * j < p.s.dim ? load8(w + (size_t)(d - dg + 16 * j) * p.s.rank) : zero8<T>();
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                float f[8];
                unpack8(v[j], f);
                const float x = d + 16 * j < p.s.dim ? qs[d + 16 * j] : 0.f;
#pragma unroll
                for (int e = 0; e < 8; ++e) acc[e] = fmaf(x, f[e], acc[e]);
            }
        }
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) part[dg][8 * (tid & 15) + e] = acc[e];
    __syncthreads();
    if (tid < 128 && r0 + tid < p.s.rank) {
        float s = 0.f;
#pragma unroll
        for (int i = 0; i < 16; ++i) s += part[i][tid];
        out[r0 + tid] = from_float<T>(s);
    }
    if (r0 == 0) {
        for (int i = tid; i < p.s.rot / 2; i += kLatThreads) {
            T *d = out + p.s.rank + 2 * i;
            if (i < p.s.rot_pairs) rotate_pair(q + p.s.dim + 2 * i, d, p.lut + ((size_t)position * p.s.rot_pairs + i) * 2);
            else d[0] = d[1] = from_float<T>(0.f);
        }
    }
}

// Rows of `chunks` times 8 elements that follow each other in memory -> LDS rows of another pitch, by the whole workgroup, in
// batches of BATCH chunks per thread: every thread requests a batch before it stores the first of it.
template <class T, int BATCH>
struct RowCopy {
    Vec8<T> v[BATCH];
    // chunks first .. of the rows at `base`; from `limit` on (past the last row) the last chunk instead
    __device__ __forceinline__ void request(const T *base, int first, int limit) {
#pragma unroll
        for (int i = 0; i < BATCH; ++i) {
            const int n = first + (int)threadIdx.x + kLatThreads * i;
            v[i] = load8(base + 8 * (n < limit ? n : limit - 1));
        }
    }
    __device__ __forceinline__ void store(T *tile, int pitch, int chunks, int first, int count) const {
        const int n0 = first + (int)threadIdx.x;
        int r = n0 / chunks, c = n0 % chunks;
        const int dr = kLatThreads / chunks, dc = kLatThreads % chunks;
#pragma unroll
        for (int i = 0; i < BATCH; ++i) {
            if (n0 + kLatThreads * i < count) store8(tile + r * pitch + 8 * c, v[i]);
            r += dr;
            c += dc;
            if (c >= chunks) {
                c -= chunks;
                ++r;
            }
        }
    }
};

// blockIdx.x = split, blockIdx.y = 16 rows (row = token * heads + head).  CT: 16-column tiles of the latent per wave.
// blockIdx.z = key / value head.  BATCH: chunks per thread that a copy of keys has in flight.
template <class T, int KB, int CT, int BATCH>
__global__ void __launch_bounds__(kLatThreads) latent_decode_kernel(const CacheView v, const T *qa, const T *cache, int M, const int32_t *pos_dev, int pos, int nsplit,
                                                                    float *part_o, float *part_ml) {
    extern __shared__ __attribute__((aligned(16))) char latent_lds[];
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int ql = lane & 15, g = lane >> 4;
    const int lq = v.q_len, row_len = v.row_len, qpitch = lq + 16 / (int)sizeof(T), pitch = row_len + 16 / (int)sizeof(T);
    const int rows = M * v.heads, row0 = blockIdx.y * 16;
    qa += (size_t)blockIdx.z * rows * lq;
    cache += (size_t)blockIdx.z * v.head_stride;
    part_o += (size_t)blockIdx.z * rows * nsplit * v.v_cols;
    part_ml += (size_t)blockIdx.z * rows * nsplit * 2;
    constexpr int SP = KB + 4, PP = KB + 8;       // pitches of the scores and of the probabilities
    T *tile = reinterpret_cast<T *>(latent_lds);  // [KB][pitch]
    T *qt = tile + KB * pitch;                    // [16][qpitch]
    T *pt = qt + 16 * qpitch;                     // [16][PP]
    float *st = reinterpret_cast<float *>(pt + 16 * PP);   // [parts][16][SP]
    float *al = st + 4 / (KB / 16) * 16 * SP;     // [16] rescaling factors of the block

    const int pos0 = pos_dev ? pos_dev[0] : pos, total = pos0 + M;
    const int first_key = first_block_key(pos0, v.window, KB);
    const int per = keys_per_split(total - first_key, nsplit, KB);
    const int k0 = first_key + blockIdx.x * per;
    const int last_row = row0 + 15 < rows ? row0 + 15 : rows - 1;
    const int seen = pos0 + last_row / v.heads + 1;            // keys that any of these rows sees
    const int k1 = k0 + per < seen ? k0 + per : seen;

    const int chunks = row_len / 8, qchunks = lq / 8;
    // A block of keys that is one batch travels to registers while the block before it is multiplied.
    RowCopy<T, BATCH> copy;
    const int count = KB * chunks;
    const bool one_batch = count <= BATCH * kLatThreads;
    // (a ring holds whole blocks: its rows of one block follow each other)
    auto request = [&](int kb, int first) {
        copy.request(cache + (size_t)(v.ring ? kb % v.ring : kb) * row_len, first, (total - kb < KB ? total - kb : KB) * chunks);
    };
    if (k0 < k1) {
        if (one_batch) request(k0, 0);
        constexpr int QB = sizeof(T) == 2 ? 5 : 3;
        RowCopy<T, QB> queries;
        const int n = 16 * qchunks, valid = (rows - row0 < 16 ? rows - row0 : 16) * qchunks;
        for (int first = 0; first < n; first += QB * kLatThreads) {
            queries.request(qa + (size_t)row0 * lq, first, valid);
            queries.store(qt, qpitch, qchunks, first, n);
        }
    }
    // softmax threads: row tid / 16, keys (tid % 16) + 16 j of a block
    const int srow = tid >> 4, skey = tid & 15;
    const int row_of_mine = row0 + srow < rows ? row0 + srow : rows - 1;
    const int my_limit = pos0 + row_of_mine / v.heads;         // last visible key ...
    const int my_first = my_limit - v.window;                  // ... and the last one in front of its window
    float m = kAttnNegBig, l = 0.f;
    floatx4 o[CT];
#pragma unroll
    for (int c = 0; c < CT; ++c) o[c] = floatx4{0.f, 0.f, 0.f, 0.f};
    const int tiles = v.v_cols / 16;
    const float scale2 = v.scale * 1.4426950408889634f;

    for (int kb = k0; kb < k1; kb += KB) {
        if (one_batch) {
            copy.store(tile, pitch, chunks, 0, count);
        } else {
            for (int first = 0; first < count; first += BATCH * kLatThreads) {
                request(kb, first);
                copy.store(tile, pitch, chunks, first, count);
            }
        }
        __syncthreads();
        if (one_batch && kb + KB < k1) request(kb + KB, 0);
        {   // 16 keys per wave; with fewer key tiles than waves, several waves share one and each takes a part of the length
            constexpr int PARTS = 4 / (KB / 16);
            const int kt = wave % (KB / 16), part = wave / (KB / 16);
            floatx4 s0 = floatx4{0.f, 0.f, 0.f, 0.f}, s1 = s0;
            const T *a = tile + (16 * kt + ql) * pitch + 8 * g, *b = qt + ql * qpitch + 8 * g;
            const int steps = lq / 32, ks1 = steps * (part + 1) / PARTS;
            int ks = steps * part / PARTS;
            for (; ks + 2 <= ks1; ks += 2) {
                s0 = mma32(load8(a + 32 * ks), load8(b + 32 * ks), s0);
                s1 = mma32(load8(a + 32 * ks + 32), load8(b + 32 * ks + 32), s1);
            }
            if (ks < ks1) s0 = mma32(load8(a + 32 * ks), load8(b + 32 * ks), s0);
            s0 += s1;
            *reinterpret_cast<floatx4 *>(st + part * 16 * SP + ql * SP + 16 * kt + 4 * g) = s0;   // keys 4 g .. of row ql
        }
        __syncthreads();
        {
            float sc[KB / 16];
            float top = kAttnNegBig;
#pragma unroll
            for (int j = 0; j < KB / 16; ++j) {
                const int key = skey + 16 * j;
                float raw = st[srow * SP + key];
#pragma unroll
                for (int q = 1; q < 4 / (KB / 16); ++q) raw += st[q * 16 * SP + srow * SP + key];
                sc[j] = kb + key <= my_limit && kb + key > my_first ? raw * scale2 : kAttnNegBig;
                top = fmaxf(top, sc[j]);
            }
            top = row_reduce16<true>(top);
            const float mn = fmaxf(m, top), alpha = __builtin_amdgcn_exp2f(m - mn);
            float sum = 0.f;
#pragma unroll
            for (int j = 0; j < KB / 16; ++j) {
                const float e = sc[j] > 0.5f * kAttnNegBig ? __builtin_amdgcn_exp2f(sc[j] - mn) : 0.f;
                sum += e;
                pt[srow * PP + skey + 16 * j] = from_float<T>(e);
            }
            l = l * alpha + row_sum16(sum);
            m = mn;
            if (skey == 0) al[srow] = alpha;
        }
        __syncthreads();
        const float alpha = al[ql];
        Vec8<T> pv[KB / 32];
#pragma unroll
        for (int t = 0; t < KB / 32; ++t) {
            float a[4], b[4];
            load4(pt + ql * PP + 32 * t + 4 * g, a);
            load4(pt + ql * PP + 32 * t + 16 + 4 * g, b);
            pv[t] = pair8<T>(floatx4{a[0], a[1], a[2], a[3]}, floatx4{b[0], b[1], b[2], b[3]});
        }
#pragma unroll
        for (int c = 0; c < CT; ++c) {
            const int ct = wave + 4 * c;
            if (ct < tiles) {
                o[c] *= alpha;
#pragma unroll
                for (int t = 0; t < KB / 32; ++t) o[c] = mma32(column8(tile + 32 * t * pitch, pitch, v.v_off + 16 * ct), pv[t], o[c]);
            }
        }
        __syncthreads();
    }
    if (k0 >= total) return;       // (the merge does not look at splits that start behind the last key)
    if (row0 + ql < rows) {
        float *dst = part_o + ((size_t)(row0 + ql) * nsplit + blockIdx.x) * v.v_cols + 4 * g;
#pragma unroll
        for (int c = 0; c < CT; ++c) {
            const int ct = wave + 4 * c;
            if (ct < tiles) *reinterpret_cast<floatx4 *>(dst + 16 * ct) = o[c];
        }
    }
    if (skey == 0 && row0 + srow < rows) {
        float *ml = part_ml + ((size_t)(row0 + srow) * nsplit + blockIdx.x) * 2;
        ml[0] = m;
        ml[1] = l;
    }
}

constexpr int kMaxSplits = 256, kValueRows = 16;
constexpr int kMergeThreads = 512, kMergeWaves = kMergeThreads / 64, kRowsPerWave = kValueRows / kMergeWaves;

// blockIdx.x = head * blocks of 16 value rows, blockIdx.y = token
template <class T>
__global__ void __launch_bounds__(kMergeThreads) latent_combine_kernel(const LatentArgs<T> p, int nsplit, int kb, const float *part_o, const float *part_ml,
                                                                     const float *sink, const T *w_uv, T *out, long ldo, int value_blocks) {
    __shared__ float f[kMaxSplits];
    __shared__ float red[2 * kMergeWaves];
    extern __shared__ __attribute__((aligned(16))) float merged[];   // [rank up to a multiple of 512], then [3][512]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int h = blockIdx.x / value_blocks, v0 = (blockIdx.x % value_blocks) * kValueRows, m = blockIdx.y;
    const size_t row = (size_t)m * p.s.heads + h;
    const int total = first_position(p) + p.M, per = keys_per_split(total, nsplit, kb);
    const int active = (total + per - 1) / per;
    const int rank = p.s.rank;

    // the first 512 columns of this wave's value rows are requested before anything is waited for
    const T *w_row = w_uv + ((size_t)h * p.s.vdim + v0 + kRowsPerWave * wave) * rank;
    Vec8<T> w_first[kRowsPerWave];
#pragma unroll
    for (int i = 0; i < kRowsPerWave; ++i) w_first[i] = 8 * lane < rank ? load8(w_row + (size_t)i * rank + 8 * lane) : zero8<T>();
    // factors of the splits in the log2 domain; the sink is one more term of the denominator
    const float snk = sink[h] * 1.4426950408889634f;
    float ms = kAttnNegBig, ls = 0.f;
    if (tid < active) {
        const float *ml = part_ml + (row * nsplit + tid) * 2;
        ms = ml[0];
        ls = ml[1];
    }
    float top = wave_reduce<true>(ms);
    if (lane == 0) red[wave] = top;
    __syncthreads();
    top = snk;
#pragma unroll
    for (int i = 0; i < kMergeWaves; ++i) top = fmaxf(top, red[i]);
    const float fac = tid < active ? exp2f(ms - top) : 0.f;
    const float part = wave_reduce<false>(fac * ls);
    if (lane == 0) red[kMergeWaves + wave] = part;
    __syncthreads();
    float den = exp2f(snk - top);
#pragma unroll
    for (int i = 0; i < kMergeWaves; ++i) den += red[kMergeWaves + i];
    if (tid < kMaxSplits) f[tid] = fac / den;
    __syncthreads();
    // merged latent: a thread adds every fourth split of four columns, the quarters meet in LDS
    const int quarter = tid >> 7, col = 4 * (tid & 127);
    float *piece = merged + (rank + 511) / 512 * 512;
    constexpr int BATCH = 16;
    for (int r0 = 0; r0 < rank; r0 += 512) {
        const int r = r0 + col;
        floatx4 s = floatx4{0.f, 0.f, 0.f, 0.f};
        if (r < rank) {
            const float *src = part_o + row * nsplit * rank + r;
            for (int i = quarter; i < active; i += 4 * BATCH) {
                floatx4 v[BATCH];
#pragma unroll
                for (int j = 0; j < BATCH; ++j) v[j] = *reinterpret_cast<const floatx4 *>(src + (size_t)(i + 4 * j < active ? i + 4 * j : i) * rank);
#pragma unroll
                for (int j = 0; j < BATCH; ++j) s += v[j] * (i + 4 * j < active ? f[i + 4 * j] : 0.f);
            }
        }
        if (quarter > 0) *reinterpret_cast<floatx4 *>(piece + 512 * (quarter - 1) + col) = s;
        __syncthreads();
        if (quarter == 0) {
#pragma unroll
            for (int q = 0; q < 3; ++q) s += *reinterpret_cast<const floatx4 *>(piece + 512 * q + col);
            *reinterpret_cast<floatx4 *>(merged + r) = s;
        }
        __syncthreads();
    }
    float mine = 0.f;
#pragma unroll
    for (int i = 0; i < kRowsPerWave; ++i) {
        float acc = 0.f;
        for (int k = 8 * lane; k < rank; k += 512) {
            float wf[8];
            unpack8(k < 512 ? w_first[i] : load8(w_row + (size_t)i * rank + k), wf);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc = fmaf(wf[e], merged[k + e], acc);
        }
        acc = wave_reduce<false>(acc);
        mine = lane == i ? acc : mine;
    }
    if (lane < kRowsPerWave) {
        const int v = h * p.s.vdim + v0 + kRowsPerWave * wave + lane;
        const float gate = to_float(p.proj[(size_t)m * p.ld + p.gate_off + v]);
        out[(size_t)m * ldo + v] = from_float<T>(mine * sigmoid_f32(gate));
    }
}

template <class T>
LatentArgs<T> args_of(const LatentShape &s, const LatentRows &r) {
    LatentArgs<T> a;
    a.s = s;
    a.proj = static_cast<const T *>(r.proj);
    a.ld = r.ld;
    a.kv_off = r.kv_off;
    a.gate_off = r.gate_off;
    a.lut = r.lut;
    a.kv_norm = r.kv_norm;
    a.eps = r.eps;
    a.cache = static_cast<T *>(r.cache);
    a.M = r.M;
    a.pos_dev = r.pos_dev;
    a.pos = r.pos;
    return a;
}

CacheView view_of(const LatentShape &s) {
    CacheView v;
    v.heads = s.heads;
    v.q_len = v.row_len = s.rank + s.rot;
    v.v_off = 0;
    v.v_cols = s.rank;
    v.scale = s.scale;
    return v;
}

template <class T>
size_t decode_lds(const CacheView &v, int kb) {
    const size_t pad = 16 / sizeof(T);
    return (kb * (v.row_len + pad) + 16 * (v.q_len + pad) + 16 * (kb + 8)) * sizeof(T) + (64 / kb * 16 * (kb + 4) + 16) * sizeof(float);
}
constexpr size_t kLdsLimit = 160 * 1024;

template <class T>
constexpr int decode_block() { return 32; }

// keys per block: fewer where a block of the usual size does not fit in LDS (0: not at all)
template <class T>
int decode_kb(const CacheView &v) {
    if (v.v_cols > 1024) return 0;
    int kb = decode_block<T>();
    while (kb >= 32 && decode_lds<T>(v, kb) > kLdsLimit) kb /= 2;
    return kb >= 32 ? kb : 0;
}

template <class T>
hipError_t decode(const CacheView &v, const void *qa, const void *cache, int M, const int32_t *pos_dev, int pos, int nsplit, float *part_o,
                  float *part_ml, hipStream_t stream) {
    const int kb = decode_kb<T>(v);
    const size_t lds = decode_lds<T>(v, kb);
    const dim3 grid(nsplit, (M * v.heads + 15) / 16, v.kv_heads);
    auto run = [&](auto kernel) {
        if (lds > 48 * 1024) {
            const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
            if (e != hipSuccess) return e;
        }
        hipLaunchKernelGGL(kernel, grid, dim3(kLatThreads), lds, stream, v, static_cast<const T *>(qa), static_cast<const T *>(cache), M, pos_dev, pos, nsplit,
                           part_o, part_ml);
        return hipGetLastError();
    };
    const int ct = (v.v_cols / 16 + 3) / 4;
    constexpr int B = sizeof(T) == 2 ? 10 : 8, S = sizeof(T) == 2 ? 4 : 8;   // short rows: a block is at most 4 (or 8) chunks per thread
    if (kb == 32) {
        if (ct <= 2 && kb * v.row_len <= 8 * S * kLatThreads) return run(&latent_decode_kernel<T, 32, 2, S>);
        if (ct <= 2) return run(&latent_decode_kernel<T, 32, 2, B>);
        if (ct <= 4) return run(&latent_decode_kernel<T, 32, 4, B>);
        if (ct <= 8) return run(&latent_decode_kernel<T, 32, 8, B>);
        return run(&latent_decode_kernel<T, 32, 16, B>);
    }
    return hipErrorInvalidValue;
}

template <class T>
hipError_t absorb(const LatentShape &s, const LatentRows &r, const void *w_uk, void *qa, hipStream_t stream) {
    const int blocks = (s.rank + 127) / 128;
    const dim3 grid(s.heads * blocks + (r.kv_off >= 0), r.M);
    hipLaunchKernelGGL(latent_absorb_kernel<T>, grid, dim3(kLatThreads), 0, stream, args_of<T>(s, r), static_cast<const T *>(w_uk), static_cast<T *>(qa),
                       blocks);
    return hipGetLastError();
}

template <class T>
hipError_t combine(const LatentShape &s, const LatentRows &r, int nsplit, const float *part_o, const float *part_ml, const float *sink, const void *w_uv,
                   void *out, long ldo, hipStream_t stream) {
    const int blocks = (s.vdim + kValueRows - 1) / kValueRows;
    hipLaunchKernelGGL(latent_combine_kernel<T>, dim3(s.heads * blocks, r.M), dim3(kMergeThreads), ((size_t)(s.rank + 511) / 512 * 512 + 3 * 512) * sizeof(float),
                       stream, args_of<T>(s, r), nsplit, decode_kb<T>(view_of(s)), part_o, part_ml, sink, static_cast<const T *>(w_uv), static_cast<T *>(out), ldo,
                       blocks);
    return hipGetLastError();
}

}  // namespace

int decode_block_keys(int dtype, const CacheView &v) { return dtype == kF32 ? decode_kb<float>(v) : decode_kb<bf16>(v); }

hipError_t launch_cache_decode(int dtype, const CacheView &v, const void *q, const void *cache, int M, const int32_t *pos_dev, int pos, int nsplit,
                               float *part_o, float *part_ml, hipStream_t stream) {
    return dtype == kF32 ? decode<float>(v, q, cache, M, pos_dev, pos, nsplit, part_o, part_ml, stream)
                         : decode<bf16>(v, q, cache, M, pos_dev, pos, nsplit, part_o, part_ml, stream);
}

bool latent_decode_supported(int dtype, const LatentShape &s) {
    return s.dim <= 1024 && decode_block_keys(dtype, view_of(s)) != 0;
}

hipError_t launch_latent_prepare(int dtype, const LatentShape &s, const LatentRows &r, hipStream_t stream) {
    if (dtype == kF32) hipLaunchKernelGGL(latent_prepare_kernel<float>, dim3(r.M), dim3(kLatThreads), 0, stream, args_of<float>(s, r));
    else hipLaunchKernelGGL(latent_prepare_kernel<bf16>, dim3(r.M), dim3(kLatThreads), 0, stream, args_of<bf16>(s, r));
    return hipGetLastError();
}

hipError_t launch_latent_absorb(int dtype, const LatentShape &s, const LatentRows &r, const void *w_uk, void *qa, hipStream_t stream) {
    return dtype == kF32 ? absorb<float>(s, r, w_uk, qa, stream) : absorb<bf16>(s, r, w_uk, qa, stream);
}

hipError_t launch_latent_decode(int dtype, const LatentShape &s, const LatentRows &r, const void *qa, int nsplit, float *part_o, float *part_ml,
                                hipStream_t stream) {
    return launch_cache_decode(dtype, view_of(s), qa, r.cache, r.M, r.pos_dev, r.pos, nsplit, part_o, part_ml, stream);
}

hipError_t launch_latent_combine(int dtype, const LatentShape &s, const LatentRows &r, int nsplit, const float *part_o, const float *part_ml,
                                 const float *sink, const void *w_uv, void *out, long ldo, hipStream_t stream) {
    return dtype == kF32 ? combine<float>(s, r, nsplit, part_o, part_ml, sink, w_uv, out, ldo, stream)
                         : combine<bf16>(s, r, nsplit, part_o, part_ml, sink, w_uv, out, ldo, stream);
}

}  // namespace w4a16
