// Row operations around the sublayers of a decoder with an fp32 residual stream and norms on
// both sides of every sublayer. Memory-bound: every tensor is read and written once.
//
//   residual_norm   x <- x + m * LN(y) * w_post, then h = LN(x) * w_pre: the norm after a
//                   sublayer, the residual sum and the norm before the next sublayer in one pass
//   embed_norm      x <- table[token], h = LN(x) * w_pre
//   silu_mul        h = silu(gate) * up
//   gated_rms_norm  out = rms_norm(o) * w * sigmoid(g)
//
// LN is the layer norm with a weight and no bias. One workgroup per token row, the row in
// registers, means and variances in two passes over the registers, all in fp32.
#include "mix_common.cuh"
#include "mix_launchers.h"

namespace astrai_mix {

namespace {

// NV > 0: the row sits in NV registers of four per thread (width % 4 == 0, width <= 1024 NV).
// NV == 0: any width, scalar accesses, x_out is the storage between the passes (a thread reads
// back only what it wrote).
template <typename T, int NV, bool EMBED>
__global__ __launch_bounds__(kRowThreads) void residual_norm_kernel(ResidualNormArgs a) {
    __shared__ float slots[kRowThreads / kWave];
    const int64_t row = blockIdx.x;
    const int w = a.width, tid = threadIdx.x;
    const float inv_w = 1.0f / (float)w;
    float* xo = a.x_out + row * w;
    T* h = static_cast<T*>(a.h) + row * w;
    const T* y = nullptr;
    if constexpr (EMBED) {
        int64_t tok = a.tokens[row];
        tok = tok < 0 ? 0 : (tok >= a.vocab ? a.vocab - 1 : tok);
        y = static_cast<const T*>(a.y) + tok * w;
    } else {
        y = static_cast<const T*>(a.y) + row * w;
    }
    const float* xi = EMBED ? nullptr : a.x_in + row * w;

    if constexpr (NV > 0) {
        f32x4 v[NV];
        float s = 0.0f;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * kRowThreads + tid) * 4;
            v[i] = c < w ? Elem<T>::get4(y + c) : f32x4{0, 0, 0, 0};
            s += (v[i][0] + v[i][1]) + (v[i][2] + v[i][3]);
        }
        if constexpr (!EMBED) {
            f32x4 x[NV];
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int c = (i * kRowThreads + tid) * 4;
                x[i] = c < w ? *reinterpret_cast<const f32x4*>(xi + c) : f32x4{0, 0, 0, 0};
            }
            const float mean = block_sum(s, slots) * inv_w;
            float q = 0.0f;
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int c = (i * kRowThreads + tid) * 4;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    v[i][e] = c < w ? v[i][e] - mean : 0.0f;
                    q += v[i][e] * v[i][e];
                }
            }
            const float r = a.mult / sqrtf(block_sum(q, slots) * inv_w + a.eps);
            s = 0.0f;
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int c = (i * kRowThreads + tid) * 4;
                if (c < w) {
                    const f32x4 g = *reinterpret_cast<const f32x4*>(a.w_post + c);
#pragma unroll
                    for (int e = 0; e < 4; ++e) v[i][e] = x[i][e] + v[i][e] * r * g[e];
                    s += (v[i][0] + v[i][1]) + (v[i][2] + v[i][3]);
                }
            }
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * kRowThreads + tid) * 4;
            if (c < w) *reinterpret_cast<f32x4*>(xo + c) = v[i];
        }
        const float mean = block_sum(s, slots) * inv_w;
        float q = 0.0f;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * kRowThreads + tid) * 4;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                v[i][e] = c < w ? v[i][e] - mean : 0.0f;
                q += v[i][e] * v[i][e];
            }
        }
        const float r = 1.0f / sqrtf(block_sum(q, slots) * inv_w + a.eps);
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * kRowThreads + tid) * 4;
            if (c < w) {
                const f32x4 g = *reinterpret_cast<const f32x4*>(a.w_pre + c);
                f32x4 o;
#pragma unroll
                for (int e = 0; e < 4; ++e) o[e] = v[i][e] * r * g[e];
                Elem<T>::put4(h + c, o);
            }
        }
    } else {
        float mean = 0.0f, r = 0.0f, s = 0.0f, q = 0.0f;
        if constexpr (!EMBED) {
            for (int c = tid; c < w; c += kRowThreads) s += Elem<T>::get(y + c);
            mean = block_sum(s, slots) * inv_w;
            for (int c = tid; c < w; c += kRowThreads) {
                const float d = Elem<T>::get(y + c) - mean;
                q += d * d;
            }
            r = a.mult / sqrtf(block_sum(q, slots) * inv_w + a.eps);
        }
        s = q = 0.0f;
        for (int c = tid; c < w; c += kRowThreads) {
            float v = Elem<T>::get(y + c);
            if constexpr (!EMBED) v = xi[c] + (v - mean) * r * a.w_post[c];
            xo[c] = v;
            s += v;
        }
        mean = block_sum(s, slots) * inv_w;
        for (int c = tid; c < w; c += kRowThreads) {
            const float d = xo[c] - mean;
            q += d * d;
        }
        r = 1.0f / sqrtf(block_sum(q, slots) * inv_w + a.eps);
        for (int c = tid; c < w; c += kRowThreads) Elem<T>::put(h + c, (xo[c] - mean) * r * a.w_pre[c]);
    }
}

template <typename T, bool EMBED>
void residual_norm_t(const ResidualNormArgs& a, hipStream_t stream) {
    const dim3 grid((unsigned)a.rows), block(kRowThreads);
    const int w = a.width;
    if (w % 4 != 0 || w > 8192) residual_norm_kernel<T, 0, EMBED><<<grid, block, 0, stream>>>(a);
    else if (w <= 1024) residual_norm_kernel<T, 1, EMBED><<<grid, block, 0, stream>>>(a);
    else if (w <= 2048) residual_norm_kernel<T, 2, EMBED><<<grid, block, 0, stream>>>(a);
    else if (w <= 4096) residual_norm_kernel<T, 4, EMBED><<<grid, block, 0, stream>>>(a);
    else residual_norm_kernel<T, 8, EMBED><<<grid, block, 0, stream>>>(a);
}

// gu [rows, 2 ff] (gate, then up), h [rows, ff]; ff % 8 == 0
template <typename T>
__global__ __launch_bounds__(256) void silu_mul_kernel(const T* gu, T* h, int64_t rows, int ff) {
    const int per_row = ff / 8;
    const int64_t total = rows * per_row;
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
        const int64_t row = i / per_row;
        const int c = (int)(i - row * per_row) * 8;
        const T* g = gu + row * 2 * ff + c;
        const f32x4 g0 = Elem<T>::get4(g), g1 = Elem<T>::get4(g + 4);
        const f32x4 u0 = Elem<T>::get4(g + ff), u1 = Elem<T>::get4(g + ff + 4);
        f32x4 o0, o1;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            o0[e] = silu_as<T>(g0[e]) * u0[e];
            o1[e] = silu_as<T>(g1[e]) * u1[e];
        }
        T* o = h + row * ff + c;
        Elem<T>::put4(o, o0);
        Elem<T>::put4(o + 4, o1);
    }
}

// o [rows, n], g rows of stride ldg, weight [n]; the mean of squares is over `count` of the n
// columns (the rest are zero padding); n % 4 == 0
template <typename T>
__global__ __launch_bounds__(kRowThreads) void gated_rms_norm_kernel(const T* o, const T* g, int64_t ldg,
                                                                     const float* w, T* out, int n, int count,
                                                                     float eps) {
    __shared__ float slots[kRowThreads / kWave];
    const int64_t row = blockIdx.x;
    o += row * n;
    g += row * ldg;
    out += row * n;
    float s = 0.0f;
    for (int c = threadIdx.x * 4; c < n; c += kRowThreads * 4) {
        const f32x4 v = Elem<T>::get4(o + c);
        s += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
    }
    const float r = 1.0f / sqrtf(block_sum(s, slots) / (float)count + eps);
    for (int c = threadIdx.x * 4; c < n; c += kRowThreads * 4) {
        const f32x4 v = Elem<T>::get4(o + c), z = Elem<T>::get4(g + c);
        const f32x4 ww = *reinterpret_cast<const f32x4*>(w + c);
        f32x4 t;
#pragma unroll
        for (int e = 0; e < 4; ++e) t[e] = v[e] * r * ww[e] * sigmoid(z[e]);
        Elem<T>::put4(out + c, t);
    }
}

}  // namespace

void launch_residual_norm(const ResidualNormArgs& a, int dtype, hipStream_t stream) {
    if (dtype) {
        if (a.tokens) residual_norm_t<float, true>(a, stream);
        else residual_norm_t<float, false>(a, stream);
    } else {
        if (a.tokens) residual_norm_t<uint16_t, true>(a, stream);
        else residual_norm_t<uint16_t, false>(a, stream);
    }
}

void launch_silu_mul(const void* gu, void* h, int64_t rows, int ff, int dtype, hipStream_t stream) {
    const int64_t blocks = (rows * (ff / 8) + 255) / 256;
    const dim3 grid((unsigned)(blocks < 8192 ? blocks : 8192));
    if (dtype)
        silu_mul_kernel<float><<<grid, 256, 0, stream>>>(static_cast<const float*>(gu), static_cast<float*>(h), rows, ff);
    else
        silu_mul_kernel<uint16_t><<<grid, 256, 0, stream>>>(static_cast<const uint16_t*>(gu),
                                                            static_cast<uint16_t*>(h), rows, ff);
}

void launch_gated_rms_norm(const void* o, const void* g, int64_t ldg, const float* w, void* out, int64_t rows,
                           int n, int count, float eps, int dtype, hipStream_t stream) {
    const dim3 grid((unsigned)rows);
    if (dtype)
        gated_rms_norm_kernel<float><<<grid, kRowThreads, 0, stream>>>(
            static_cast<const float*>(o), static_cast<const float*>(g), ldg, w, static_cast<float*>(out), n, count, eps);
    else
        gated_rms_norm_kernel<uint16_t><<<grid, kRowThreads, 0, stream>>>(
            static_cast<const uint16_t*>(o), static_cast<const uint16_t*>(g), ldg, w, static_cast<uint16_t*>(out), n,
            count, eps);
}

}  // namespace astrai_mix
