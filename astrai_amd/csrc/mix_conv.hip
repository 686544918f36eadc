// Short causal convolution per channel, with the last inputs of every sequence kept in a ring.
//
//   conv       out_t = act(bias + sum_j w_j x_(t - taps + 1 + j)); inputs before the block come from the ring
//   conv_tail  the block's last taps - 1 inputs into the ring. Its own launch: a block may be longer than the
//              ring, whose rows other workgroups of conv still read
#include "mix_conv.cuh"
#include "mix_launchers.h"

namespace astrai_mix {

namespace {

constexpr int kStrip = 8;   // tokens per thread

// a thread: four channels of kStrip consecutive tokens; TAPS > 0: the inputs slide through registers
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void conv_kernel(ConvArgs a) {
    const int quads = a.cols / 4, strips = (a.seq + kStrip - 1) / kStrip;
    const int64_t item = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (item >= (int64_t)quads * strips * a.batch) return;
    const int c = (int)(item % quads) * 4;
    const int64_t rest = item / quads;
    const int t0 = (int)(rest % strips) * kStrip, b = (int)(rest / strips);
    const int t1 = min(t0 + kStrip, a.seq);
    const int64_t start = a.positions[0];
    const f32x4 bias = a.bias ? *reinterpret_cast<const f32x4*>(a.bias + c) : f32x4{0, 0, 0, 0};
    auto finish = [&](int t, f32x4 s) {
        if (a.silu) {
#pragma unroll
            for (int e = 0; e < 4; ++e) s[e] = silu_as<T>(s[e]);
        }
        Elem<T>::put4(static_cast<T*>(a.out) + ((int64_t)b * a.seq + t) * a.cols + c, s);
    };
    if constexpr (TAPS > 0) {
        f32x4 w[TAPS], x[TAPS];
#pragma unroll
        for (int j = 0; j < TAPS; ++j) w[j] = *reinterpret_cast<const f32x4*>(a.taps_w + (int64_t)j * a.cols + c);
#pragma unroll
        for (int j = 1; j < TAPS; ++j) x[j] = conv_input4<T>(a, b, start, t0 - TAPS + j, c);
#pragma unroll
        for (int i = 0; i < kStrip; ++i) {
            const int t = t0 + i;
            if (t < t1) {
#pragma unroll
                for (int j = 0; j + 1 < TAPS; ++j) x[j] = x[j + 1];
                x[TAPS - 1] = conv_input4<T>(a, b, start, t, c);
                f32x4 s = bias;
#pragma unroll
                for (int j = 0; j < TAPS; ++j)
#pragma unroll
                    for (int e = 0; e < 4; ++e) s[e] = fmaf(x[j][e], w[j][e], s[e]);
                finish(t, s);
            }
        }
    } else {
        for (int t = t0; t < t1; ++t) finish(t, conv_at4<T>(a, b, start, t, c));
    }
}

template <typename T>
__global__ __launch_bounds__(256) void conv_tail_kernel(ConvArgs a) {
    const int quads = a.cols / 4, n = min(a.taps - 1, a.seq);
    const int64_t item = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (item >= (int64_t)quads * n * a.batch) return;
    const int64_t rest = item / quads;
    ring_put4<T>(a, (int)(rest / n), a.positions[0], a.seq - n + (int)(rest % n), (int)(item % quads) * 4);
}

template <typename T>
void conv_t(const ConvArgs& a, hipStream_t stream) {
    const int64_t items = (int64_t)(a.cols / 4) * ((a.seq + kStrip - 1) / kStrip) * a.batch;
    const dim3 grid((unsigned)((items + 255) / 256));
    if (a.taps == 2) conv_kernel<T, 2><<<grid, 256, 0, stream>>>(a);
    else if (a.taps == 3) conv_kernel<T, 3><<<grid, 256, 0, stream>>>(a);
    else if (a.taps == 4) conv_kernel<T, 4><<<grid, 256, 0, stream>>>(a);
    else conv_kernel<T, 0><<<grid, 256, 0, stream>>>(a);
}

}  // namespace

void launch_conv(const ConvArgs& a, int dtype, hipStream_t stream) {
    if (dtype) conv_t<float>(a, stream);
    else conv_t<uint16_t>(a, stream);
}

void launch_conv_tail(const ConvArgs& a, int dtype, hipStream_t stream) {
    const int n = a.taps - 1 < a.seq ? a.taps - 1 : a.seq;
    if (n == 0) return;
    const int64_t items = (int64_t)(a.cols / 4) * n * a.batch;
    const dim3 grid((unsigned)((items + 255) / 256));
    if (dtype) conv_tail_kernel<float><<<grid, 256, 0, stream>>>(a);
    else conv_tail_kernel<uint16_t><<<grid, 256, 0, stream>>>(a);
}

}  // namespace astrai_mix
