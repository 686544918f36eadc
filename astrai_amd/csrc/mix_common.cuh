// Pieces shared by the kernels of libastrai_mix.so (sequence mixers and row operations of
// models with an fp32 residual stream): element access for the two activation types, the
// two-term bf16 split that carries a 32-bit factor through the bf16 matrix cores, and the
// transposing LDS read.
#pragma once

#include "common.cuh"
#include "row_ops.cuh"

namespace astrai_mix {

using w8a8::block_sum;
using w8a8::f32_to_bf16;
using w8a8::f32x2;
using w8a8::f32x4;
using w8a8::kRowThreads;
using w8a8::kWave;
using w8a8::pack_bf16x2;
using w8a8::u32x2;
using w8a8::u32x4;

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef short i16x4 __attribute__((ext_vector_type(4)));

constexpr float kNegBig = -1e30f;  // finite stand-in for -inf: no inf - inf
constexpr float kLog2e = 1.44269504088896340736f;

// Activation types: bf16 (as raw 16-bit words) and float.
template <typename T>
struct Elem;

template <>
struct Elem<uint16_t> {
    static __device__ __forceinline__ float get(const uint16_t* p) { return w8a8::bf16_to_f32(*p); }
    static __device__ __forceinline__ void put(uint16_t* p, float v) { *p = f32_to_bf16(v); }
    static __device__ __forceinline__ f32x4 get4(const uint16_t* p) {
        const u32x2 r = *reinterpret_cast<const u32x2*>(p);
        return f32x4{__uint_as_float(r.x << 16), __uint_as_float(r.x & 0xffff0000u),
                     __uint_as_float(r.y << 16), __uint_as_float(r.y & 0xffff0000u)};
    }
    static __device__ __forceinline__ void put4(uint16_t* p, f32x4 v) {
        *reinterpret_cast<u32x2*>(p) = u32x2{pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3])};
    }
};

template <>
struct Elem<float> {
    static __device__ __forceinline__ float get(const float* p) { return *p; }
    static __device__ __forceinline__ void put(float* p, float v) { *p = v; }
    static __device__ __forceinline__ f32x4 get4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
    static __device__ __forceinline__ void put4(float* p, f32x4 v) { *reinterpret_cast<f32x4*>(p) = v; }
};

__device__ __forceinline__ float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu(float z) { return z / (1.0f + expf(-z)); }

// the same on the hardware exponential and reciprocal, for results that are rounded to bf16
__device__ __forceinline__ float silu_fast(float z) {
    return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-kLog2e * z));
}

template <typename T>
__device__ __forceinline__ float silu_as(float z) {
    return sizeof(T) == 2 ? silu_fast(z) : silu(z);
}

// tanh as 1 - 2 / (1 + e^(2z)), absolute error about 1e-7; e^(2z) may overflow or vanish
__device__ __forceinline__ float tanh_fast(float z) {
    return 1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(2.0f * kLog2e * z));
}

__device__ __forceinline__ float sigmoid_fast(float z) {
    return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-kLog2e * z));
}

// gelu in its tanh form, z / 2 (1 + tanh(y)) = z sigmoid(2 y), y = sqrt(2 / pi) (z + 0.044715 z^3)
template <typename T>
__device__ __forceinline__ float gelu_as(float z) {
    const float y2 = 1.5957691216057308f * (z + 0.044715f * z * z * z);
    return z * (sizeof(T) == 2 ? sigmoid_fast(y2) : sigmoid(y2));
}

// log(1 + e^z): max(z, 0) + log(1 + e), e = e^-|z| in (0, 1]; a Taylor polynomial for small e, where 1 + e
// would drop its digits
__device__ __forceinline__ float softplus_fast(float z) {
    const float e = __builtin_amdgcn_exp2f(-kLog2e * fabsf(z));
    const float big = 0.69314718055994530942f * __builtin_amdgcn_logf(1.0f + e);
    float p = 1.0f / 6.0f;
    p = 1.0f / 5.0f - e * p;
    p = 1.0f / 4.0f - e * p;
    p = 1.0f / 3.0f - e * p;
    p = 1.0f / 2.0f - e * p;
    p = e * (1.0f - e * p);
    return fmaxf(z, 0.0f) + (e < 0.0625f ? p : big);
}

template <typename T>
__device__ __forceinline__ float softplus_as(float z) {
    return sizeof(T) == 2 ? softplus_fast(z) : fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z)));
}

// silu of eight bf16 values, rounded to bf16
__device__ __forceinline__ u32x4 silu8_bf16(u32x4 raw) {
    float f[8];
    w8a8::unpack8(raw, f);
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] = silu_fast(f[e]);
    return u32x4{pack_bf16x2(f[0], f[1]), pack_bf16x2(f[2], f[3]), pack_bf16x2(f[4], f[5]),
                 pack_bf16x2(f[6], f[7])};
}

// x = hi + lo to 2^-17 of |x|, both bf16: two bf16 MFMAs then multiply by a 32-bit factor
__device__ __forceinline__ void split2(float a, float b, uint32_t& hi, uint32_t& lo) {
    hi = pack_bf16x2(a, b);
    lo = pack_bf16x2(a - __uint_as_float(hi << 16), b - __uint_as_float(hi & 0xffff0000u));
}

__device__ __forceinline__ f32x4 mfma16(u32x4 a, u32x4 b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a),
                                                   __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}

__device__ __forceinline__ f32x16 mfma32(u32x4 a, u32x4 b, f32x16 c) {
    return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, a),
                                                   __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}

// Transposing LDS read. In each 16-lane group, lane 4j+q points at row j, columns 4q..4q+3 of a
// 4-row x 16-column patch of 16-bit values and receives column (its index in the group) of
// rows 0..3. Two of them make the eight contraction positions of one MFMA operand register set.
__device__ __forceinline__ u32x2 lds_read_tr(const uint8_t* src) {
    typedef __attribute__((address_space(3))) i16x4 lds_i16x4;
    return __builtin_bit_cast(u32x2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(src)));
}

__device__ __forceinline__ u32x4 join(u32x2 a, u32x2 b) { return u32x4{a.x, a.y, b.x, b.y}; }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int off = 32; off; off >>= 1) v += __shfl_xor(v, off, kWave);
    return v;
}

}  // namespace astrai_mix
