// Row operations around the sublayers of a decoder with an fp32 residual stream and norms on
// both sides of every sublayer. Memory-bound: every tensor is read and written once.
//
//   residual_norm   x <- x + m * LN(y) * w_post, then h = LN(x) * w_pre: the norm after a
//                   sublayer, the residual sum and the norm before the next sublayer in one pass
//   embed_norm      x <- table[token], h = LN(x) * w_pre
//   sum_norm        x <- the sum of up to four terms, then h = RMS(x) * w: the residual sum and the norm
//                   before the next sublayer, or a stream that is begun anew
//   act_mul         h = act(gate) * up
//   gated_rms_norm  out = rms_norm(o) * w * sigmoid(g), over a row or over each head of it
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

// x <- mult * (table[token] or y) + x_in + u + vec, each but the first optional; h = x / sqrt(mean(x^2) + eps) * w,
// or x itself without w. TY: type of y and u. NV as above.
template <typename T, typename TY, int NV>
__global__ __launch_bounds__(kRowThreads) void sum_norm_kernel(SumNormArgs a) {
    __shared__ float slots[kRowThreads / kWave];
    const int64_t row = blockIdx.x;
    const int w = a.width, tid = threadIdx.x;
    int64_t src = row;
    if (a.tokens) {
        src = a.tokens[row];
        src = src < 0 ? 0 : (src >= a.vocab ? a.vocab - 1 : src);
    }
    const TY* y = static_cast<const TY*>(a.y) + src * a.ldy;
    const TY* u = a.u ? static_cast<const TY*>(a.u) + row * a.ldu : nullptr;
    const float* xi = a.x_in ? a.x_in + row * w : nullptr;
    float* xo = a.x_out + row * w;
    T* h = static_cast<T*>(a.h) + row * w;
    if constexpr (NV > 0) {
        f32x4 v[NV];
        float s = 0.0f;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * kRowThreads + tid) * 4;
            v[i] = f32x4{0, 0, 0, 0};
            if (c < w) {
                v[i] = Elem<TY>::get4(y + c);
#pragma unroll
                for (int e = 0; e < 4; ++e) v[i][e] *= a.mult;
                if (xi) v[i] += *reinterpret_cast<const f32x4*>(xi + c);
                if (u) v[i] += Elem<TY>::get4(u + c);
                if (a.vec) v[i] += *reinterpret_cast<const f32x4*>(a.vec + c);
                *reinterpret_cast<f32x4*>(xo + c) = v[i];
            }
            s += (v[i][0] * v[i][0] + v[i][1] * v[i][1]) + (v[i][2] * v[i][2] + v[i][3] * v[i][3]);
        }
        float r = 1.0f;
        if (a.w) r = 1.0f / sqrtf(block_sum(s, slots) / (float)w + a.eps);
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = (i * kRowThreads + tid) * 4;
            if (c < w) {
                f32x4 o = v[i];
                if (a.w) {
                    const f32x4 g = *reinterpret_cast<const f32x4*>(a.w + c);
#pragma unroll
                    for (int e = 0; e < 4; ++e) o[e] = v[i][e] * r * g[e];
                }
                Elem<T>::put4(h + c, o);
            }
        }
    } else {
        float s = 0.0f, r = 1.0f;
        for (int c = tid; c < w; c += kRowThreads) {
            float v = Elem<TY>::get(y + c) * a.mult;
            if (xi) v += xi[c];
            if (u) v += Elem<TY>::get(u + c);
            if (a.vec) v += a.vec[c];
            xo[c] = v;
            s += v * v;
        }
        if (a.w) r = 1.0f / sqrtf(block_sum(s, slots) / (float)w + a.eps);
        for (int c = tid; c < w; c += kRowThreads) Elem<T>::put(h + c, a.w ? xo[c] * r * a.w[c] : xo[c]);
    }
}

template <typename T, typename TY>
void sum_norm_t(const SumNormArgs& a, hipStream_t stream) {
    const dim3 grid((unsigned)a.rows), block(kRowThreads);
    const int w = a.width;
    if (w % 4 != 0 || a.ldy % 4 != 0 || a.ldu % 4 != 0 || w > 8192) sum_norm_kernel<T, TY, 0><<<grid, block, 0, stream>>>(a);
    else if (w <= 1024) sum_norm_kernel<T, TY, 1><<<grid, block, 0, stream>>>(a);
    else if (w <= 2048) sum_norm_kernel<T, TY, 2><<<grid, block, 0, stream>>>(a);
    else if (w <= 4096) sum_norm_kernel<T, TY, 4><<<grid, block, 0, stream>>>(a);
    else sum_norm_kernel<T, TY, 8><<<grid, block, 0, stream>>>(a);
}

// gu [rows, 2 ff] (gate, then up), h [rows, ff]; ff % 8 == 0
template <typename T, int ACT>
__device__ __forceinline__ float act_as(float z) {
    return ACT == kActGelu ? gelu_as<T>(z) : silu_as<T>(z);
}

template <typename T, int ACT>
__global__ __launch_bounds__(256) void act_mul_kernel(const T* gu, T* h, int64_t rows, int ff) {
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
            o0[e] = act_as<T, ACT>(g0[e]) * u0[e];
            o1[e] = act_as<T, ACT>(g1[e]) * u1[e];
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

// the same over each head's vp columns (count of them real): `lanes` threads per (row, head)
template <typename T>
__global__ __launch_bounds__(256) void head_gated_rms_norm_kernel(HeadNormArgs a, int lanes) {
    const int64_t item = (int64_t)blockIdx.x * (256 / lanes) + threadIdx.x / lanes;
    const int lane = threadIdx.x % lanes;
    const bool live = item < a.rows * a.heads;
    const int64_t row = live ? item / a.heads : 0, at = live ? item * a.vp : 0;
    const T* o = static_cast<const T*>(a.o) + at;
    const T* g = static_cast<const T*>(a.g) + row * a.ldg + (live ? item - row * a.heads : 0) * a.vp;
    T* out = static_cast<T*>(a.out) + at;
    float s = 0.0f;
    for (int c = lane * 4; c < a.vp; c += lanes * 4) {
        const f32x4 v = Elem<T>::get4(o + c);
        s += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
    }
    for (int off = lanes / 2; off; off >>= 1) s += __shfl_xor(s, off, kWave);
    if (!live) return;
    const float r = 1.0f / sqrtf(s / (float)a.count + a.eps);
    for (int c = lane * 4; c < a.vp; c += lanes * 4) {
        const f32x4 v = Elem<T>::get4(o + c), z = Elem<T>::get4(g + c);
        const f32x4 w = *reinterpret_cast<const f32x4*>(a.w + c);
        f32x4 t;
#pragma unroll
        for (int e = 0; e < 4; ++e) t[e] = v[e] * r * w[e] * sigmoid(z[e]);
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

void launch_sum_norm(const SumNormArgs& a, int dtype, bool y_float, hipStream_t stream) {
    if (dtype) sum_norm_t<float, float>(a, stream);
    else if (y_float) sum_norm_t<uint16_t, float>(a, stream);
    else sum_norm_t<uint16_t, uint16_t>(a, stream);
}

void launch_act_mul(const void* gu, void* h, int64_t rows, int ff, int act, int dtype, hipStream_t stream) {
    const int64_t blocks = (rows * (ff / 8) + 255) / 256;
    const dim3 grid((unsigned)(blocks < 8192 ? blocks : 8192));
    auto run = [&](auto zero) {
        using T = decltype(zero);
        const T* in = static_cast<const T*>(gu);
        T* out = static_cast<T*>(h);
        if (act == kActGelu) act_mul_kernel<T, kActGelu><<<grid, 256, 0, stream>>>(in, out, rows, ff);
        else act_mul_kernel<T, kActSilu><<<grid, 256, 0, stream>>>(in, out, rows, ff);
    };
    if (dtype) run(float{});
    else run(uint16_t{});
}

void launch_head_gated_rms_norm(const HeadNormArgs& a, int dtype, hipStream_t stream) {
    int lanes = 8;   // per head: a power of two, four columns each
    while (lanes < 64 && lanes * 4 < a.vp) lanes *= 2;
    const int64_t items = a.rows * a.heads, per = 256 / lanes;
    const dim3 grid((unsigned)((items + per - 1) / per));
    if (dtype) head_gated_rms_norm_kernel<float><<<grid, 256, 0, stream>>>(a, lanes);
    else head_gated_rms_norm_kernel<uint16_t><<<grid, 256, 0, stream>>>(a, lanes);
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
