// Real-gated linear recurrent unit behind a short convolution, per channel
//   r, i = sigmoid(W_r u + b_r), sigmoid(W_i u + b_i)   (block-diagonal W)
//   a = exp(coef r),  S <- a S + sqrt(1 - a^2) i u,  out = S gelu(y)
// with coef = -8 softplus(lam). Gates, decays and the state are fp32.
//
// Chunk kernel (prompts, bf16). A workgroup takes one block of channels (or a part of its outputs) and a
// segment of one sequence, and walks it in tiles of 16 NT tokens. The tile of u sits in LDS; a wave
// forms both gate products of 16 channels on v_mfma_f32_16x16x32_bf16 with tokens as rows, so that a lane
// holds four consecutive tokens of one channel and the recurrence is a scan: four steps in the lane, two
// exchanges between the four lanes of a channel, and the state carried from tile to tile.
// With few workgroups the sequence is cut into segments that run side by side: one pass forms every
// segment's decay and contribution, the output pass folds those of the segments before its own.
//
// Step kernel (decoding, bf16): convolution, both products, recurrence and output gate in one launch; a
// workgroup takes 16 channels of 16 rows (sequences x new tokens), its waves share out the block's inputs.
//
// General path (any block size, bf16 or float): gates per element, then the recurrence token by token.
#include "mix_conv.cuh"
#include "mix_launchers.h"

namespace astrai_mix {

namespace {

struct Decay {
    float a, b;   // S <- a S + b
};

// log a = coef r <= 0
__device__ __forceinline__ Decay decay_exact(float zr, float zi, float coef, float u) {
    const float log_a = coef * sigmoid(zr);
    return Decay{expf(log_a), sqrtf(-expm1f(2.0f * log_a)) * sigmoid(zi) * u};
}

// The same on the hardware's exponential, reciprocal and root, of sums without their biases: b = -log2(e) bias,
// coef2 = log2(e) coef, so that e = log2 a and 1 - a^2 = 1 - 2^(2 e), a Taylor polynomial in e where the difference
// would cancel.
__device__ __forceinline__ Decay decay_fast(float sr, float br, float si, float bi, float coef2, float u) {
    const float r = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(fmaf(sr, -kLog2e, br)));
    const float i = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(fmaf(si, -kLog2e, bi)));
    const float e = coef2 * r;
    Decay d;
    d.a = __builtin_amdgcn_exp2f(e);
    constexpr float c = 1.38629436111989061883f;   // 2 ln 2
    float p = fmaf(e, c / 5.0f, 1.0f);
    p = fmaf(e * (c / 4.0f), p, 1.0f);
    p = fmaf(e * (c / 3.0f), p, 1.0f);
    p = fmaf(e * (c / 2.0f), p, 1.0f);
    const float m = e > -0.07f ? -c * e * p : fmaf(-d.a, d.a, 1.0f);
    d.b = __builtin_amdgcn_sqrtf(m) * i * u;
    return d;
}

__device__ __forceinline__ float gelu_fast(float z) {   // gelu_as with log2(e) in its constants
    constexpr float c = -kLog2e * 1.5957691216057308f;
    const float t = z * fmaf(z * z, c * 0.044715f, c);
    return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(t));
}

template <int NT, bool OUT>
__global__ __launch_bounds__(256, 3) void rglru_chunk_kernel(RglruArgs a, int csplit) {
    constexpr int kTile = NT * 16;
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    const int bp = a.bp, row_bytes = bp * 2 + 16;
    float* carry_s = reinterpret_cast<float*>(lds + kTile * row_bytes);   // [bp]: a channel belongs to one wave
    float* carry_a = carry_s + bp;
    const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int seg = blockIdx.x, blk = (int)blockIdx.y / csplit, part = (int)blockIdx.y % csplit, b = blockIdx.z;
    const int cols = a.blocks * bp;
    const int tiles = (a.seq + kTile - 1) / kTile, per_seg = (tiles + a.nseg - 1) / a.nseg;
    const int tok0 = min(seg * per_seg * kTile, a.seq), tok1 = min((seg + 1) * per_seg * kTile, a.seq);
    const bool last = seg == a.nseg - 1;
    // scratch [batch, nseg, 2, cols]: decay and contribution of a segment; the last one's slot keeps the
    // state the block starts from
    auto slot = [&](int s, int which) { return a.scratch + (((int64_t)b * a.nseg + s) * 2 + which) * cols + blk * bp; };
    float* state = a.state + (int64_t)b * cols + blk * bp;

    for (int ct = part * 4 + wave; ct < bp / 16; ct += 4 * csplit) {
        const int ch = ct * 16 + c16;
        if (g == 0) {
            float s = 0.0f;
            if constexpr (OUT) {
                if (a.nseg == 1) {
                    s = state[ch];
                } else {
                    s = slot(a.nseg - 1, 1)[ch];
                    for (int j = 0; j < seg; ++j) s = fmaf(slot(j, 0)[ch], s, slot(j, 1)[ch]);
                }
            } else if (last) {
                slot(seg, 1)[ch] = state[ch];
            }
            carry_s[ch] = s;
            carry_a[ch] = 1.0f;
        }
    }
    if (!OUT && last) return;

    const uint16_t* u = static_cast<const uint16_t*>(a.u) + (int64_t)b * a.seq * cols + blk * bp;
    const int c8 = bp / 8, row0 = tid / c8, e0 = tid % c8, row_step = 256 / c8, e_step = 256 % c8;
    for (int t0 = tok0; t0 < tok1; t0 += kTile) {
        __syncthreads();   // the previous tile is no longer read; the carries are there
        // (eight loads in flight; a thread's chunks are 256 apart)
        for (int row = row0, e = e0; row < kTile;) {
            u32x4 v[8];
            int at[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                at[j] = row < kTile ? row * row_bytes + e * 16 : -1;
                const int t = t0 + row;
                v[j] = u32x4{0, 0, 0, 0};
                if (row < kTile && t < tok1) v[j] = *reinterpret_cast<const u32x4*>(u + (int64_t)t * cols + e * 8);
                row += row_step;
                e += e_step;
                if (e >= c8) {
                    e -= c8;
                    ++row;
                }
            }
#pragma unroll
            for (int j = 0; j < 8; ++j)
                if (at[j] >= 0) *reinterpret_cast<u32x4*>(lds + at[j]) = v[j];
        }
        __syncthreads();
        const int left = min(tok1 - t0, kTile);
        for (int ct = part * 4 + wave; ct < bp / 16; ct += 4 * csplit) {
            const int ch = ct * 16 + c16, col = blk * bp + ch;
            // the output gates' inputs, asked for ahead of the products (past the end: the last token's)
            uint16_t yv[OUT ? NT : 1][4];
            // (buffer descriptors end with the segment: later tokens read as 0 and are not written)
            const __amdgpu_buffer_rsrc_t ry = w8a8::make_rsrc(
                static_cast<const uint16_t*>(a.proj) + ((int64_t)b * a.seq + t0) * a.ld, (uint32_t)(left * a.ld) * 2);
            const __amdgpu_buffer_rsrc_t ro = w8a8::make_rsrc(
                static_cast<const uint16_t*>(a.out) + ((int64_t)b * a.seq + t0) * cols, (uint32_t)(left * cols) * 2);
            const uint32_t y_lane = (uint32_t)(4 * g * a.ld + a.y_off + col) * 2, o_lane = (uint32_t)(4 * g * cols + col) * 2;
            if constexpr (OUT) {
#pragma unroll
                for (int tt = 0; tt < NT; ++tt)
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        yv[tt][e] = __builtin_amdgcn_raw_buffer_load_b16(ry, y_lane + (uint32_t)((tt * 16 + e) * a.ld) * 2, 0, 0);
            }
            f32x4 zr[NT], zi[NT];
#pragma unroll
            for (int tt = 0; tt < NT; ++tt) zr[tt] = zi[tt] = f32x4{0, 0, 0, 0};
            const int64_t w_row = ((int64_t)blk * bp + ch) * bp + 8 * g;
            const uint16_t* wr = static_cast<const uint16_t*>(a.w_r) + w_row;
            const uint16_t* wi = static_cast<const uint16_t*>(a.w_i) + w_row;
            const uint8_t* lu = lds + c16 * row_bytes + 16 * g;
            // weight operands two steps ahead
            u32x4 fr = *reinterpret_cast<const u32x4*>(wr), fi = *reinterpret_cast<const u32x4*>(wi);
            const int k1 = bp > 32 ? 32 : 0;
            u32x4 mr = *reinterpret_cast<const u32x4*>(wr + k1), mi = *reinterpret_cast<const u32x4*>(wi + k1);
            for (int k = 0; k < bp; k += 32) {
                const int kn = k + 64 < bp ? k + 64 : k;
                const u32x4 nr = *reinterpret_cast<const u32x4*>(wr + kn), ni = *reinterpret_cast<const u32x4*>(wi + kn);
#pragma unroll
                for (int tt = 0; tt < NT; ++tt) {
                    const u32x4 x = *reinterpret_cast<const u32x4*>(lu + tt * 16 * row_bytes + k * 2);
                    zr[tt] = mfma16(x, fr, zr[tt]);
                    zi[tt] = mfma16(x, fi, zi[tt]);
                }
                fr = mr;
                fi = mi;
                mr = nr;
                mi = ni;
            }
            const float br = -kLog2e * a.b_r[col], bi = -kLog2e * a.b_i[col], coef2 = kLog2e * a.coef[col];
            float s_in = carry_s[ch], a_in = carry_a[ch];
#pragma unroll
            for (int tt = 0; tt < NT; ++tt) {
                const int tl = tt * 16 + 4 * g;   // this lane's first token in the tile
                Decay d[4];
                float pa = 1.0f, pb = 0.0f;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float x = w8a8::bf16_to_f32(
                        *reinterpret_cast<const uint16_t*>(lds + (tl + e) * row_bytes + ch * 2));
                    d[e] = decay_fast(zr[tt][e], br, zi[tt][e], bi, coef2, x);
                }
                if (left < kTile) {
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (tl + e >= left) d[e] = Decay{1.0f, 0.0f};
                }
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    pa *= d[e].a;
                    pb = fmaf(d[e].a, pb, d[e].b);
                }
                // over the lane groups: inclusive, then what comes before this lane
                float qa = __shfl_up(pa, 16, kWave), qb = __shfl_up(pb, 16, kWave);
                if (g >= 1) {
                    pb = fmaf(pa, qb, pb);
                    pa *= qa;
                }
                qa = __shfl_up(pa, 32, kWave);
                qb = __shfl_up(pb, 32, kWave);
                if (g >= 2) {
                    pb = fmaf(pa, qb, pb);
                    pa *= qa;
                }
                const float xa = __shfl_up(pa, 16, kWave), xb = __shfl_up(pb, 16, kWave);
                float s = g ? fmaf(xa, s_in, xb) : s_in;
                const float ta = __shfl(pa, 48 + c16, kWave), tb = __shfl(pb, 48 + c16, kWave);
                s_in = fmaf(ta, s_in, tb);
                a_in *= ta;
                if constexpr (OUT) {
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        s = fmaf(d[e].a, s, d[e].b);
                        const float o = s * gelu_fast(w8a8::bf16_to_f32(yv[tt][e]));
                        __builtin_amdgcn_raw_buffer_store_b16(f32_to_bf16(o), ro, o_lane + (uint32_t)((tt * 16 + e) * cols) * 2, 0, 0);
                    }
                }
            }
            if (g == 0) {   // (every group has read the carries: the wave's lanes run together)
                carry_s[ch] = s_in;
                carry_a[ch] = a_in;
            }
        }
    }
    __syncthreads();
    for (int ct = part * 4 + wave; ct < bp / 16; ct += 4 * csplit) {
        const int ch = ct * 16 + c16;
        if (g == 0) {
            if constexpr (!OUT) {
                slot(seg, 0)[ch] = carry_a[ch];
                slot(seg, 1)[ch] = carry_s[ch];
            } else if (last) {
                state[ch] = carry_s[ch];
            }
        }
    }
}

// rows: a workgroup's sequences b0 .. b0 + nb - 1, seq tokens each, nb * seq <= 16
__global__ __launch_bounds__(256) void rglru_step_kernel(RglruArgs a, int nb) {
    __shared__ f32x4 red[3][2][64];
    __shared__ float zs[2][16][17];
    __shared__ float us[16][17];   // the convolved inputs of this workgroup's channels
    const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int bp = a.bp, per = bp / 16, cols = a.blocks * bp;
    const int blk = (int)blockIdx.x / per, ct = (int)blockIdx.x % per;
    const int b0 = (int)blockIdx.y * nb, n_seq = min(nb, a.batch - b0), n_live = n_seq * a.seq;
    const int64_t start = a.conv.positions[0];
    // for the recurrence a thread takes one channel of one sequence; what it needs is asked for now
    const int ch = tid & 15, col = blk * bp + ct * 16 + ch, bl = tid >> 4;
    const bool mine = bl < n_seq;
    const int b = b0 + (mine ? bl : 0);
    const uint16_t* y_src = static_cast<const uint16_t*>(a.proj) + (int64_t)b * a.seq * a.ld + a.y_off + col;
    float s = a.state[(int64_t)b * cols + col];
    const float coef2 = kLog2e * a.coef[col], br = -kLog2e * a.b_r[col], bi = -kLog2e * a.b_i[col];
    uint16_t y_next = y_src[0];
    {
        const int row = min(c16, n_live - 1), rb = b0 + row / a.seq, t = row % a.seq;
        const int64_t w_row = ((int64_t)blk * bp + ct * 16 + c16) * bp;
        f32x4 zr = {0, 0, 0, 0}, zi = {0, 0, 0, 0};
        for (int k = wave * 32 + 8 * g; k < bp; k += 128) {
            const u32x4 fr = *reinterpret_cast<const u32x4*>(static_cast<const uint16_t*>(a.w_r) + w_row + k);
            const u32x4 fi = *reinterpret_cast<const u32x4*>(static_cast<const uint16_t*>(a.w_i) + w_row + k);
            const f32x4 x0 = conv_at4<uint16_t>(a.conv, rb, start, t, blk * bp + k);
            const f32x4 x1 = conv_at4<uint16_t>(a.conv, rb, start, t, blk * bp + k + 4);
            const u32x4 x = {pack_bf16x2(x0[0], x0[1]), pack_bf16x2(x0[2], x0[3]), pack_bf16x2(x1[0], x1[1]),
                             pack_bf16x2(x1[2], x1[3])};
            if (k / 16 == ct) {
                float f[8];
                w8a8::unpack8(x, f);
#pragma unroll
                for (int e = 0; e < 8; ++e) us[c16][k % 16 + e] = f[e];
            }
            zr = mfma16(x, fr, zr);
            zi = mfma16(x, fi, zi);
        }
        if (wave) {
            red[wave - 1][0][lane] = zr;
            red[wave - 1][1][lane] = zi;
        }
        __syncthreads();
        if (wave == 0) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                zs[0][4 * g + e][c16] = (zr[e] + red[0][0][lane][e]) + (red[1][0][lane][e] + red[2][0][lane][e]);
                zs[1][4 * g + e][c16] = (zi[e] + red[0][1][lane][e]) + (red[1][1][lane][e] + red[2][1][lane][e]);
            }
        }
        __syncthreads();
    }
    if (!mine) return;
    for (int t = 0; t < a.seq; ++t) {
        const int r = bl * a.seq + t;
        const float y = w8a8::bf16_to_f32(y_next);
        if (t + 1 < a.seq) y_next = y_src[(int64_t)(t + 1) * a.ld];
        const Decay d = decay_fast(zs[0][r][ch], br, zs[1][r][ch], bi, coef2, us[r][ch]);
        s = fmaf(d.a, s, d.b);
        Elem<uint16_t>::put(static_cast<uint16_t*>(a.out) + ((int64_t)b * a.seq + t) * cols + col, s * gelu_fast(y));
    }
    a.state[(int64_t)b * cols + col] = s;
    // this block's last inputs into the ring: rows that no workgroup of this launch reads
    if (ch % 4 == 0)
        for (int t = max(a.seq - a.conv.taps + 1, 0); t < a.seq; ++t) ring_put4<uint16_t>(a.conv, b, start, t, col);
}

// a thread per (token, channel); w_r, w_i are [blocks, in, out]
template <typename T>
__global__ __launch_bounds__(256) void rglru_gates_kernel(RglruArgs a) {
    const int cols = a.blocks * a.bp;
    const int64_t tokens = (int64_t)a.batch * a.seq, item = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (item >= tokens * cols) return;
    const int col = (int)(item % cols), blk = col / a.bp, ch = col - blk * a.bp;
    const T* u = static_cast<const T*>(a.u) + item - ch;
    const T* wr = static_cast<const T*>(a.w_r) + (int64_t)blk * a.bp * a.bp + ch;
    const T* wi = static_cast<const T*>(a.w_i) + (int64_t)blk * a.bp * a.bp + ch;
    float zr = 0.0f, zi = 0.0f;
    for (int k = 0; k < a.bp; ++k) {
        const float x = Elem<T>::get(u + k);
        zr = fmaf(x, Elem<T>::get(wr + (int64_t)k * a.bp), zr);
        zi = fmaf(x, Elem<T>::get(wi + (int64_t)k * a.bp), zi);
    }
    const Decay d = decay_exact(zr + a.b_r[col], zi + a.b_i[col], a.coef[col], Elem<T>::get(u + ch));
    a.scratch[item] = d.a;
    a.scratch[tokens * cols + item] = d.b;
}

template <typename T>
__global__ __launch_bounds__(64) void rglru_scan_kernel(RglruArgs a) {
    const int cols = a.blocks * a.bp;
    const int col = (int)blockIdx.x * 64 + threadIdx.x, b = blockIdx.y;
    if (col >= cols) return;
    float s = a.state[(int64_t)b * cols + col];
    const int64_t tokens = (int64_t)a.batch * a.seq;
    for (int t = 0; t < a.seq; ++t) {
        const int64_t row = (int64_t)b * a.seq + t, at = row * cols + col;
        s = fmaf(a.scratch[at], s, a.scratch[tokens * cols + at]);
        const float y = Elem<T>::get(static_cast<const T*>(a.proj) + row * a.ld + a.y_off + col);
        Elem<T>::put(static_cast<T*>(a.out) + at, s * gelu_as<T>(y));
    }
    a.state[(int64_t)b * cols + col] = s;
}

template <int NT>
void chunk_t(const RglruArgs& a, hipStream_t stream) {
    const int shared = NT * 16 * (a.bp * 2 + 16) + 2 * a.bp * (int)sizeof(float);
    static const hipError_t once = [] {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&rglru_chunk_kernel<NT, true>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        return e != hipSuccess ? e : hipFuncSetAttribute(reinterpret_cast<const void*>(&rglru_chunk_kernel<NT, false>),
                                                         hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    }();
    (void)once;
    // parts of a block's outputs: until there are about two workgroups per CU, each wave keeping a tile
    const int most = (a.bp + 63) / 64;
    int csplit = 1;
    while (csplit < most && (int64_t)a.nseg * a.blocks * a.batch * csplit < 512) ++csplit;
    const dim3 grid((unsigned)a.nseg, (unsigned)(a.blocks * csplit), (unsigned)a.batch);
    if (a.nseg > 1) rglru_chunk_kernel<NT, false><<<grid, 256, shared, stream>>>(a, csplit);
    rglru_chunk_kernel<NT, true><<<grid, 256, shared, stream>>>(a, csplit);
}

template <typename T>
void general_t(const RglruArgs& a, hipStream_t stream) {
    const int cols = a.blocks * a.bp;
    const int64_t items = (int64_t)a.batch * a.seq * cols;
    rglru_gates_kernel<T><<<(unsigned)((items + 255) / 256), 256, 0, stream>>>(a);
    rglru_scan_kernel<T><<<dim3((unsigned)((cols + 63) / 64), (unsigned)a.batch), 64, 0, stream>>>(a);
}

}  // namespace

// a tile of 64 tokens of 1024 channels: 129 KiB of LDS, the carries 8 KiB
bool rglru_chunk_supported(int bp) { return bp <= 1024; }

void launch_rglru_chunk(const RglruArgs& a, hipStream_t stream) { chunk_t<4>(a, stream); }

bool rglru_step_supported(int bp, int seq) { return bp > 0 && seq <= kRingSteps; }

void launch_rglru_step(const RglruArgs& a, hipStream_t stream) {
    const int nb = 16 / a.seq;
    const dim3 grid((unsigned)(a.blocks * (a.bp / 16)), (unsigned)((a.batch + nb - 1) / nb));
    rglru_step_kernel<<<grid, 256, 0, stream>>>(a, nb);
}

void launch_rglru_general(const RglruArgs& a, int dtype, hipStream_t stream) {
    if (dtype) general_t<float>(a, stream);
    else general_t<uint16_t>(a, stream);
}

}  // namespace astrai_mix
