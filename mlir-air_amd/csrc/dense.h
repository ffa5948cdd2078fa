// Element types and MFMA operands of the dense-weight kernels (dense_gemv.hip, dense_gemm.hip, latent_attention.hip,
// latent_prefill.hip, moe.hip).  Every one of them exists for bf16 (bf16 operands, fp32 accumulation) and for float
// (fp32 operands and fp32 MFMA: true 32-bit products); both read eight consecutive k per lane for a step of 32 k, so
// the kernels are one template over the element type.
#pragma once

#include "common.h"

namespace w4a16 {

typedef __bf16 bf16;
typedef short shortx4 __attribute__((ext_vector_type(4)));

template <class T>
struct Vec8;
template <>
struct Vec8<bf16> {
    u32x4 v;
};
template <>
struct Vec8<float> {
    floatx4 lo, hi;
};

__device__ __forceinline__ Vec8<bf16> load8(const bf16 *p) { return {*reinterpret_cast<const u32x4 *>(p)}; }
__device__ __forceinline__ Vec8<float> load8(const float *p) {
    return {*reinterpret_cast<const floatx4 *>(p), *reinterpret_cast<const floatx4 *>(p + 4)};
}
// weights of a decode step: read once, kept out of the way of what is read again
__device__ __forceinline__ Vec8<bf16> stream8(const bf16 *p) {
    return {__builtin_nontemporal_load(reinterpret_cast<const u32x4 *>(p))};
}
__device__ __forceinline__ Vec8<float> stream8(const float *p) {
    return {__builtin_nontemporal_load(reinterpret_cast<const floatx4 *>(p)),
            __builtin_nontemporal_load(reinterpret_cast<const floatx4 *>(p + 4))};
}
__device__ __forceinline__ void store8(bf16 *p, const Vec8<bf16> &v) { *reinterpret_cast<u32x4 *>(p) = v.v; }
__device__ __forceinline__ void store8(float *p, const Vec8<float> &v) {
    *reinterpret_cast<floatx4 *>(p) = v.lo;
    *reinterpret_cast<floatx4 *>(p + 4) = v.hi;
}
template <class T>
__device__ __forceinline__ Vec8<T> zero8();
template <>
__device__ __forceinline__ Vec8<bf16> zero8<bf16>() { return {u32x4{0u, 0u, 0u, 0u}}; }
template <>
__device__ __forceinline__ Vec8<float> zero8<float>() { return {floatx4{0.f, 0.f, 0.f, 0.f}, floatx4{0.f, 0.f, 0.f, 0.f}}; }

__device__ __forceinline__ float to_float(bf16 v) { return static_cast<float>(v); }
__device__ __forceinline__ float to_float(float v) { return v; }
template <class T>
__device__ __forceinline__ T from_float(float v) { return static_cast<T>(v); }

// eight floats of a Vec8
__device__ __forceinline__ void unpack8(const Vec8<bf16> &v, float (&f)[8]) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const uint32_t w = v.v[i];
        f[2 * i] = bf16_bits_to_float(w & 0xFFFFu);
        f[2 * i + 1] = bf16_bits_to_float(w >> 16);
    }
}
__device__ __forceinline__ void unpack8(const Vec8<float> &v, float (&f)[8]) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        f[i] = v.lo[i];
        f[4 + i] = v.hi[i];
    }
}

template <class T>
__device__ __forceinline__ Vec8<T> pack8(const float (&f)[8]);
template <>
__device__ __forceinline__ Vec8<bf16> pack8<bf16>(const float (&f)[8]) {
    return {u32x4{pack_bf16x2(f[0], f[1]), pack_bf16x2(f[2], f[3]), pack_bf16x2(f[4], f[5]), pack_bf16x2(f[6], f[7])}};
}
template <>
__device__ __forceinline__ Vec8<float> pack8<float>(const float (&f)[8]) { return {floatx4{f[0], f[1], f[2], f[3]}, floatx4{f[4], f[5], f[6], f[7]}}; }

// four floats -> four consecutive elements (8 or 16 bytes, aligned)
__device__ __forceinline__ void store4(bf16 *p, float a, float b, float c, float d) {
    *reinterpret_cast<uint2 *>(p) = uint2{pack_bf16x2(a, b), pack_bf16x2(c, d)};
}
__device__ __forceinline__ void store4(float *p, float a, float b, float c, float d) {
    *reinterpret_cast<floatx4 *>(p) = floatx4{a, b, c, d};
}
__device__ __forceinline__ void load4(const bf16 *p, float (&f)[4]) {
    const uint2 w = *reinterpret_cast<const uint2 *>(p);
    f[0] = bf16_bits_to_float(w.x & 0xFFFFu);
    f[1] = bf16_bits_to_float(w.x >> 16);
    f[2] = bf16_bits_to_float(w.y & 0xFFFFu);
    f[3] = bf16_bits_to_float(w.y >> 16);
}
__device__ __forceinline__ void load4(const float *p, float (&f)[4]) {
    const floatx4 w = *reinterpret_cast<const floatx4 *>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) f[i] = w[i];
}

// acc + sum of the eight products (exact bf16 products, fp32 sums)
__device__ __forceinline__ float dot8(const Vec8<bf16> &a, const Vec8<bf16> &b, float acc) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const uint32_t x = a.v[i], y = b.v[i];   // (scalars first: a bit cast of a vector element reads element 0)
        acc = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2, x), __builtin_bit_cast(bf16x2, y), acc, false);
    }
    return acc;
}
__device__ __forceinline__ float dot8(const Vec8<float> &a, const Vec8<float> &b, float acc) {
#pragma unroll
    for (int i = 0; i < 4; ++i) acc = fmaf(a.lo[i], b.lo[i], acc);
#pragma unroll
    for (int i = 0; i < 4; ++i) acc = fmaf(a.hi[i], b.hi[i], acc);
    return acc;
}

// D[i][j] += sum over 32 k of A[i][k] B[j][k], 16 x 16.  Lane l gives row l % 16 of A and of B, k = 8 (l / 16) .. + 7, and
// holds D rows 4 (l / 16) .. + 3 of column l % 16.  (The fp32 form is eight products over k = {j, 8 + j, 16 + j, 24 + j}.)
__device__ __forceinline__ floatx4 mma32(const Vec8<bf16> &a, const Vec8<bf16> &b, floatx4 d) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a.v), __builtin_bit_cast(bf16x8, b.v), d, 0, 0, 0);
}
__device__ __forceinline__ floatx4 mma32(const Vec8<float> &a, const Vec8<float> &b, floatx4 d) {
#pragma unroll
    for (int i = 0; i < 4; ++i) d = __builtin_amdgcn_mfma_f32_16x16x4f32(a.lo[i], b.lo[i], d, 0, 0, 0);
#pragma unroll
    for (int i = 0; i < 4; ++i) d = __builtin_amdgcn_mfma_f32_16x16x4f32(a.hi[i], b.hi[i], d, 0, 0, 0);
    return d;
}

// Operand for products whose k runs over the ROWS of a row-major LDS tile (pitch in elements): lane l gets column
// col0 + l % 16 at the eight rows {4 g .. 4 g + 3, 16 + 4 g .. + 3} of the 32 rows at `tile` (g = l / 16).  A sum over
// k does not care about its order, so the other operand only has to list the same rows in the same slots
// (pair8 below).  bf16 goes through the transposing LDS read: within 16 lanes, lane i receives element i % 4 of the
// 8-byte chunks addressed by lanes i / 4, i / 4 + 4, i / 4 + 8, i / 4 + 12.
__device__ __forceinline__ Vec8<bf16> column8(const bf16 *tile, int pitch, int col0) {
    const int lane = threadIdx.x & 63, i = lane & 15, g = lane >> 4;
    const bf16 *src = tile + (4 * g + (i >> 2)) * pitch + col0 + 4 * (i & 3);
    const shortx4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) shortx4 *)src);
    const shortx4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) shortx4 *)(src + 16 * pitch));
    const uint2 l2 = __builtin_bit_cast(uint2, lo), h2 = __builtin_bit_cast(uint2, hi);
    return {u32x4{l2.x, l2.y, h2.x, h2.y}};
}
__device__ __forceinline__ Vec8<float> column8(const float *tile, int pitch, int col0) {
    const int lane = threadIdx.x & 63, i = lane & 15, g = lane >> 4;
    const float *src = tile + 4 * g * pitch + col0 + i;
    Vec8<float> v;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        v.lo[j] = src[j * pitch];
        v.hi[j] = src[(16 + j) * pitch];
    }
    return v;
}
// The matching operand from registers: a = rows 4 g .. + 3, b = rows 16 + 4 g .. + 3.
template <class T>
__device__ __forceinline__ Vec8<T> pair8(floatx4 a, floatx4 b);
template <>
__device__ __forceinline__ Vec8<bf16> pair8<bf16>(floatx4 a, floatx4 b) {
    return {u32x4{pack_bf16x2(a[0], a[1]), pack_bf16x2(a[2], a[3]), pack_bf16x2(b[0], b[1]), pack_bf16x2(b[2], b[3])}};
}
template <>
__device__ __forceinline__ Vec8<float> pair8<float>(floatx4 a, floatx4 b) { return {a, b}; }

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f32(float z) { return z / (1.0f + expf(-z)); }
// the same by the hardware's reciprocal where the result is rounded to bf16 anyway
template <class T>
__device__ __forceinline__ float sigmoid_of(float z) {
    if constexpr (sizeof(T) == 2) return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
    return sigmoid_f32(z);
}
__device__ __forceinline__ float gelu_tanh_f32(float z) { return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * fmaf(0.044715f * z * z, z, z))); }
// log(1 + e^z) = max(z, 0) + log(1 + t), t = e^-|z|; log(1 + t) = log(u) t / (u - 1) with u the rounded 1 + t, whose error the
// quotient takes back (Goldberg, "What Every Computer Scientist Should Know About Floating-Point Arithmetic", 1991)
__device__ __forceinline__ float softplus_f32(float z) {
    const float t = __builtin_amdgcn_exp2f(-1.4426950408889634f * fabsf(z)), u = 1.0f + t, d = u - 1.0f;
    const float l = 0.6931471805599453f * __builtin_amdgcn_logf(u) * t * __builtin_amdgcn_rcpf(d);
    return fmaxf(z, 0.0f) + (d == 0.0f ? t : l);
}

// sum over a group of `n` neighbouring lanes (a power of two), every lane of it receiving the sum
__device__ __forceinline__ float group_sum(float v, int n) {
    for (int m = 1; m < n; m <<= 1) v += __shfl_xor(v, m, 64);
    return v;
}

// float -> unsigned key of the same order (-0 counts as +0)
__device__ __forceinline__ uint32_t order_key(float v) {
    uint32_t b = __builtin_bit_cast(uint32_t, v);
    if (b == 0x80000000u) b = 0;
    return (b & 0x80000000u) ? ~b : (b | 0x80000000u);
}
__device__ __forceinline__ unsigned long long wave_max_u64(unsigned long long v) {
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) {
        const unsigned long long o = __shfl_xor(v, m, 64);
        v = o > v ? o : v;
    }
    return v;
}

}  // namespace w4a16
