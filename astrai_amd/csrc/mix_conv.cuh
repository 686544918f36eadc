// The short convolution's inputs: of this block from the projection, earlier ones from the ring.
#pragma once

#include "mix_common.cuh"
#include "mix_launchers.h"

namespace astrai_mix {

__device__ __forceinline__ int64_t ring_row(const ConvArgs& a, int b, int64_t p) {   // p >= 0
    return (int64_t)b * a.ring_rows + (uint32_t)p % (uint32_t)a.ring_rows;
}

// four channels of the input of token t of the block (t < 0: before it); zeros before the sequence. One load
// without a branch around it, so that several can be in flight.
template <typename T>
__device__ __forceinline__ f32x4 conv_input4(const ConvArgs& a, int b, int64_t start, int t, int c) {
    const int64_t p = start + t;
    const T* src = t >= 0 ? static_cast<const T*>(a.proj) + ((int64_t)b * a.seq + t) * a.ld + a.off
                          : static_cast<const T*>(a.ring) + ring_row(a, b, p < 0 ? 0 : p) * a.cols;
    f32x4 x = Elem<T>::get4(src + c);
    if (p < 0) x = f32x4{0, 0, 0, 0};
    return x;
}

template <typename T, int TAPS>
__device__ __forceinline__ f32x4 conv_taps4(const ConvArgs& a, int b, int64_t start, int t, int c, f32x4 s) {
    f32x4 x[TAPS], w[TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
        x[j] = conv_input4<T>(a, b, start, t - TAPS + 1 + j, c);
        w[j] = *reinterpret_cast<const f32x4*>(a.taps_w + (int64_t)j * a.cols + c);
    }
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) s[e] = fmaf(x[j][e], w[j][e], s[e]);
    return s;
}

// bias + the taps' sum, no activation
template <typename T>
__device__ __forceinline__ f32x4 conv_at4(const ConvArgs& a, int b, int64_t start, int t, int c) {
    f32x4 s = a.bias ? *reinterpret_cast<const f32x4*>(a.bias + c) : f32x4{0, 0, 0, 0};
    if (a.taps == 4) return conv_taps4<T, 4>(a, b, start, t, c, s);
    if (a.taps == 3) return conv_taps4<T, 3>(a, b, start, t, c, s);
    if (a.taps == 2) return conv_taps4<T, 2>(a, b, start, t, c, s);
    for (int j = 0; j < a.taps; ++j) {
        const f32x4 x = conv_input4<T>(a, b, start, t - a.taps + 1 + j, c);
        const f32x4 w = *reinterpret_cast<const f32x4*>(a.taps_w + (int64_t)j * a.cols + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) s[e] = fmaf(x[e], w[e], s[e]);
    }
    return s;
}

// the block's token t >= 0 into the ring
template <typename T>
__device__ __forceinline__ void ring_put4(const ConvArgs& a, int b, int64_t start, int t, int c) {
    const int64_t p = start + t;
    if (p < 0) return;
    Elem<T>::put4(static_cast<T*>(a.ring) + ring_row(a, b, p) * a.cols + c,
                  Elem<T>::get4(static_cast<const T*>(a.proj) + ((int64_t)b * a.seq + t) * a.ld + a.off + c));
}

// a value as the activation type holds it
template <typename T>
__device__ __forceinline__ float rounded(float v) {
    T tmp;
    Elem<T>::put(&tmp, v);
    return Elem<T>::get(&tmp);
}

}  // namespace astrai_mix
