// The short convolution's inputs: of this block from the projection, earlier ones from the ring.
#pragma once

#include "mix_common.cuh"
#include "mix_launchers.h"

namespace astrai_mix {

// four channels of the input of token t of the block (t < 0: before it); zeros before the sequence
template <typename T>
__device__ __forceinline__ f32x4 conv_input4(const ConvArgs& a, int b, int64_t start, int t, int c) {
    if (t >= 0) return Elem<T>::get4(static_cast<const T*>(a.proj) + ((int64_t)b * a.seq + t) * a.ld + a.off + c);
    const int64_t p = start + t;
    if (p < 0) return f32x4{0, 0, 0, 0};
    const int64_t row = (int64_t)b * a.ring_rows + (int)(p % a.ring_rows);
    return Elem<T>::get4(static_cast<const T*>(a.ring) + row * a.cols + c);
}

// bias + the taps' sum, no activation
template <typename T>
__device__ __forceinline__ f32x4 conv_at4(const ConvArgs& a, int b, int64_t start, int t, int c) {
    f32x4 s = a.bias ? *reinterpret_cast<const f32x4*>(a.bias + c) : f32x4{0, 0, 0, 0};
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
    const int64_t row = (int64_t)b * a.ring_rows + (int)(p % a.ring_rows);
    Elem<T>::put4(static_cast<T*>(a.ring) + row * a.cols + c,
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
