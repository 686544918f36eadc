// Lightning attention: per head a matrix state with a constant decay,
//   S_t = decay S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,
// q, k, v being silu of the projections (rounded to the activation type). The state is fp32.
//
// Chunk kernel (prompts, bf16). A workgroup takes one head, a slice of 32 or 64 value columns and
// a segment of the sequence, walking it in chunks of 64 tokens:
//   o_i   = decay^(i+1) S^T q_i + sum_(j <= i) decay^(i-j) (q_i . k_j) v_j
//   S_new = decay^n S + sum_j decay^(n-1-j) k_j v_j^T
// on v_mfma_f32_16x16x32_bf16, outputs transposed (value columns as rows, tokens as columns): the
// score accumulator of a wave's 16 tokens is the next product's operand layout already. Every
// 32-bit factor -- the decayed scores, the state, the decay-weighted values -- enters the matrix
// cores as two bf16 terms; the state itself stays in fp32 accumulators, wave w owning its rows
// 16 (w + 4 i) ...
//
// With few heads, a long prompt is cut into segments that run side by side: one pass forms every
// segment's own contribution to the state, a scan turns those into the state each segment starts
// from, and the output pass starts there.
//
// Step kernel (decoding, short portions, and float): token by token, the state in registers.
#include "mix_common.cuh"
#include "mix_launchers.h"

namespace astrai_mix {

namespace {

constexpr int kC = kLightningChunk;

template <int DP, int VS, bool OUT>
__global__ __launch_bounds__(256, DP <= 128 ? 2 : 1) void lightning_chunk_kernel(LightningArgs a) {
    constexpr int kKRow = DP * 2 + 16, kVRow = VS * 2 + 16, kSRow = DP * 2 + 16;   // bytes
    constexpr int ND = DP / 32;                       // score steps
    constexpr int NDT = (DP / 16 + 3) / 4;            // state row tiles of a wave
    constexpr int NVT = VS / 16;
    constexpr int KC8 = DP / 8, VC8 = VS / 8;
    constexpr int NKL = kC * KC8 / 256, NVL = (kC * VC8 + 255) / 256;
    __shared__ __attribute__((aligned(16))) uint8_t lk[kC * kKRow];
    __shared__ __attribute__((aligned(16))) uint8_t lv[OUT ? kC * kVRow : 16];
    __shared__ __attribute__((aligned(16))) uint8_t lvh[kC * kVRow];
    __shared__ __attribute__((aligned(16))) uint8_t lvl[kC * kVRow];
    __shared__ __attribute__((aligned(16))) uint8_t lsh[OUT ? VS * kSRow : 16];
    __shared__ __attribute__((aligned(16))) uint8_t lsl[OUT ? VS * kSRow : 16];
    __shared__ float pw[kC + 1];

    const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int seg = blockIdx.x, v0 = (int)blockIdx.y * VS;
    const int b = (int)blockIdx.z / a.heads, head = (int)blockIdx.z % a.heads;
    const int chunks = (a.seq + kC - 1) / kC, per_seg = (chunks + a.nseg - 1) / a.nseg;
    const int tok0 = min(seg * per_seg * kC, a.seq), tok1 = min((seg + 1) * per_seg * kC, a.seq);

    if (tid <= kC) pw[tid] = a.decay_pow[head * (kC + 1) + tid];

    const int64_t state_sz = (int64_t)a.dp * a.vp;
    float* own = a.state + ((int64_t)b * a.heads + head) * state_sz;
    float* segp = a.nseg > 1 ? a.seg_state + (((int64_t)b * a.heads + head) * a.nseg + seg) * state_sz : own;
    // state: rows d = 16 (wave + 4 i) + 4 g + e, columns v0 + 16 vt + c16
    f32x4 st[NDT][NVT];
#pragma unroll
    for (int i = 0; i < NDT; ++i)
#pragma unroll
        for (int vt = 0; vt < NVT; ++vt)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int dd = 16 * (wave + 4 * i) + 4 * g + e, v = v0 + 16 * vt + c16;
                st[i][vt][e] = (OUT && dd < a.dp && v < a.vp) ? segp[(int64_t)dd * a.vp + v] : 0.0f;
            }

    const uint16_t* base = static_cast<const uint16_t*>(a.proj) + (int64_t)b * a.seq * a.ld;
    const uint16_t* kp = base + a.k_off + head * a.dp;
    const uint16_t* vp = base + a.v_off + head * a.vp + v0;
    const uint16_t* qp = base + a.q_off + head * a.dp + 8 * g;
    const u32x4 zero = {0, 0, 0, 0};
    u32x4 rk[NKL], rv[NVL], rq[ND];
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < NKL; ++i) {
            const int c = tid + i * 256, t = t0 + c / KC8, e = (c % KC8) * 8;
            rk[i] = (t < tok1 && e < a.dp) ? *reinterpret_cast<const u32x4*>(kp + (int64_t)t * a.ld + e) : zero;
        }
#pragma unroll
        for (int i = 0; i < NVL; ++i) {
            const int c = tid + i * 256, t = t0 + c / VC8, e = (c % VC8) * 8;
            rv[i] = (c < kC * VC8 && t < tok1 && v0 + e < a.vp) ? *reinterpret_cast<const u32x4*>(vp + (int64_t)t * a.ld + e)
                                                                 : zero;
        }
        if constexpr (OUT) {
            const int t = t0 + wave * 16 + c16;
#pragma unroll
            for (int i = 0; i < ND; ++i)
                rq[i] = (t < tok1 && i * 32 + 8 * g < a.dp) ? *reinterpret_cast<const u32x4*>(qp + (int64_t)t * a.ld + i * 32)
                                                            : zero;
        }
    };
    if (tok0 < tok1) fetch(tok0);
    for (int t0 = tok0; t0 < tok1; t0 += kC) {
        const int n = min(kC, tok1 - t0);
        __syncthreads();   // the previous chunk's tiles are no longer read; pw is there
        u32x4 qf[ND];
        if constexpr (OUT) {
#pragma unroll
            for (int i = 0; i < ND; ++i) qf[i] = silu8_bf16(rq[i]);
            // the state the chunk starts from, [v][d], two terms
#pragma unroll
            for (int i = 0; i < NDT; ++i)
#pragma unroll
                for (int vt = 0; vt < NVT; ++vt) {
                    const int dd = 16 * (wave + 4 * i) + 4 * g;
                    if (dd < DP) {
                        uint32_t h0, l0, h1, l1;
                        split2(st[i][vt][0], st[i][vt][1], h0, l0);
                        split2(st[i][vt][2], st[i][vt][3], h1, l1);
                        const int off = (16 * vt + c16) * kSRow + dd * 2;
                        *reinterpret_cast<u32x2*>(lsh + off) = u32x2{h0, h1};
                        *reinterpret_cast<u32x2*>(lsl + off) = u32x2{l0, l1};
                    }
                }
        }
#pragma unroll
        for (int i = 0; i < NKL; ++i) {
            const int c = tid + i * 256;
            *reinterpret_cast<u32x4*>(lk + (c / KC8) * kKRow + (c % KC8) * 16) = silu8_bf16(rk[i]);
        }
#pragma unroll
        for (int i = 0; i < NVL; ++i) {
            const int c = tid + i * 256, j = c / VC8;
            if (c < kC * VC8) {
                const int off = j * kVRow + (c % VC8) * 16;
                const u32x4 v = silu8_bf16(rv[i]);
                if constexpr (OUT) *reinterpret_cast<u32x4*>(lv + off) = v;
                const float f = j < n ? pw[n - 1 - j] : 0.0f;
                float x[8];
                w8a8::unpack8(v, x);
                u32x4 hi, lo;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    uint32_t h2, l2;
                    split2(x[2 * e] * f, x[2 * e + 1] * f, h2, l2);
                    hi[e] = h2;
                    lo[e] = l2;
                }
                *reinterpret_cast<u32x4*>(lvh + off) = hi;
                *reinterpret_cast<u32x4*>(lvl + off) = lo;
            }
        }
        __syncthreads();
        fetch(t0 + kC);

        // transposed operands: group g supplies contraction rows 4g .. 4g+3 and 16 + 4g .. of a
        // 32-row step, the order in which the score accumulators hold their keys
        const int tr_row = 4 * g + (c16 >> 2), tr_col = (c16 & 3) * 8;
        if constexpr (OUT) {
            if (wave * 16 < n) {
                f32x4 o[NVT];
#pragma unroll
                for (int vt = 0; vt < NVT; ++vt) {
                    o[vt] = f32x4{0, 0, 0, 0};
#pragma unroll
                    for (int i = 0; i < ND; ++i) {
                        const int off = (16 * vt + c16) * kSRow + i * 64 + g * 16;
                        o[vt] = mfma16(*reinterpret_cast<const u32x4*>(lsh + off), qf[i], o[vt]);
                        o[vt] = mfma16(*reinterpret_cast<const u32x4*>(lsl + off), qf[i], o[vt]);
                    }
                }
                const int qt = wave * 16 + c16;   // this lane's token in the chunk
                const float f0 = pw[qt + 1];
#pragma unroll
                for (int vt = 0; vt < NVT; ++vt)
#pragma unroll
                    for (int e = 0; e < 4; ++e) o[vt][e] *= f0;
#pragma unroll
                for (int p = 0; p < 2; ++p) {
                    if (p * 32 <= wave * 16) {
                        u32x4 hi, lo;
#pragma unroll
                        for (int u = 0; u < 2; ++u) {
                            f32x4 s = {0, 0, 0, 0};
                            const int j0 = p * 32 + u * 16;
#pragma unroll
                            for (int i = 0; i < ND; ++i)
                                s = mfma16(*reinterpret_cast<const u32x4*>(lk + (j0 + c16) * kKRow + i * 64 + g * 16), qf[i], s);
#pragma unroll
                            for (int e = 0; e < 4; ++e) {
                                const int dist = qt - (j0 + 4 * g + e);
                                s[e] = dist >= 0 ? s[e] * pw[max(dist, 0)] : 0.0f;
                            }
                            uint32_t h0, l0, h1, l1;
                            split2(s[0], s[1], h0, l0);
                            split2(s[2], s[3], h1, l1);
                            hi[2 * u] = h0;
                            hi[2 * u + 1] = h1;
                            lo[2 * u] = l0;
                            lo[2 * u + 1] = l1;
                        }
                        const uint8_t* v = lv + (p * 32 + tr_row) * kVRow + tr_col;
#pragma unroll
                        for (int vt = 0; vt < NVT; ++vt) {
                            const u32x4 vf = join(lds_read_tr(v + vt * 32), lds_read_tr(v + vt * 32 + 16 * kVRow));
                            o[vt] = mfma16(vf, hi, o[vt]);
                            o[vt] = mfma16(vf, lo, o[vt]);
                        }
                    }
                }
                const int t = t0 + qt;
                if (t < tok1) {
                    uint16_t* out = static_cast<uint16_t*>(a.out) + (((int64_t)b * a.seq + t) * a.heads + head) * a.vp + v0;
#pragma unroll
                    for (int vt = 0; vt < NVT; ++vt)
                        if (v0 + vt * 16 < a.vp) Elem<uint16_t>::put4(out + vt * 16 + 4 * g, o[vt]);
                }
            }
        }
        // state
        const float fn = pw[n];
#pragma unroll
        for (int i = 0; i < NDT; ++i)
#pragma unroll
            for (int vt = 0; vt < NVT; ++vt)
#pragma unroll
                for (int e = 0; e < 4; ++e) st[i][vt][e] *= fn;
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            const int row = p * 32 + tr_row;
            u32x4 kf[NDT];
#pragma unroll
            for (int i = 0; i < NDT; ++i) {
                const int dt = min(wave + 4 * i, DP / 16 - 1);
                const uint8_t* k = lk + row * kKRow + dt * 32 + tr_col;
                kf[i] = join(lds_read_tr(k), lds_read_tr(k + 16 * kKRow));
            }
#pragma unroll
            for (int vt = 0; vt < NVT; ++vt) {
                const uint8_t* vh = lvh + row * kVRow + vt * 32 + tr_col;
                const uint8_t* vl = lvl + row * kVRow + vt * 32 + tr_col;
                const u32x4 fh = join(lds_read_tr(vh), lds_read_tr(vh + 16 * kVRow));
                const u32x4 fl = join(lds_read_tr(vl), lds_read_tr(vl + 16 * kVRow));
#pragma unroll
                for (int i = 0; i < NDT; ++i) {
                    st[i][vt] = mfma16(kf[i], fh, st[i][vt]);
                    st[i][vt] = mfma16(kf[i], fl, st[i][vt]);
                }
            }
        }
    }
    // one segment: the state of the sequence; else this segment's own contribution to it
    if (!OUT || a.nseg == 1) {
#pragma unroll
        for (int i = 0; i < NDT; ++i)
#pragma unroll
            for (int vt = 0; vt < NVT; ++vt)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int dd = 16 * (wave + 4 * i) + 4 * g + e, v = v0 + 16 * vt + c16;
                    if (dd < a.dp && v < a.vp) segp[(int64_t)dd * a.vp + v] = st[i][vt][e];
                }
    }
}

// contributions of the segments -> the state each one starts from; the sequence's state moves on
// by the whole block. One thread per state element.
__global__ __launch_bounds__(256) void lightning_scan_kernel(LightningArgs a) {
    const int64_t sz = (int64_t)a.dp * a.vp;
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= sz) return;
    const int64_t bh = blockIdx.y;
    const int head = (int)(bh % a.heads);
    const int chunks = (a.seq + kC - 1) / kC, per_seg = (chunks + a.nseg - 1) / a.nseg;
    const float* pw = a.decay_pow + head * (kC + 1);
    float full = 1.0f;   // decay over a whole segment
    for (int c = 0; c < per_seg; ++c) full *= pw[kC];
    float* seg = a.seg_state + bh * a.nseg * sz + i;
    float s = a.state[bh * sz + i];
    for (int k = 0; k < a.nseg; ++k) {
        const int t0 = min(k * per_seg * kC, a.seq), n = min((k + 1) * per_seg * kC, a.seq) - t0;
        float f = full;
        if (n < per_seg * kC) {
            f = pw[n % kC];
            for (int c = 0; c < n / kC; ++c) f *= pw[kC];
        }
        const float u = seg[(int64_t)k * sz];
        seg[(int64_t)k * sz] = s;
        s = f * s + u;
    }
    a.state[bh * sz + i] = s;
}

// Token by token. One workgroup per (32 value columns, head, sequence): lane % 8 owns four value
// columns, the other 32 (lane / 8, wave) combinations own state rows d = r + 32 i.
template <typename T, int ND>
__global__ __launch_bounds__(256) void lightning_step_kernel(LightningArgs a) {
    __shared__ float red[2][4][32];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int v = (int)blockIdx.x * 32 + (lane & 7) * 4, r = wave * 8 + (lane >> 3);
    const int head = blockIdx.y, b = blockIdx.z;
    float* state = a.state + ((int64_t)b * a.heads + head) * a.dp * a.vp + v;
    const float decay = a.decay_pow[head * (kC + 1) + 1];
    const int nd = a.dp / 32;
    f32x4 s[ND];
#pragma unroll
    for (int i = 0; i < ND; ++i)
        s[i] = i < nd ? *reinterpret_cast<const f32x4*>(state + (int64_t)(r + 32 * i) * a.vp) : f32x4{0, 0, 0, 0};
    for (int t = 0; t < a.seq; ++t) {
        const T* row = static_cast<const T*>(a.proj) + ((int64_t)b * a.seq + t) * a.ld;
        const T* q = row + a.q_off + head * a.dp + r;
        const T* k = row + a.k_off + head * a.dp + r;
        auto act = [](float z) {
            T tmp;
            Elem<T>::put(&tmp, silu_as<T>(z));
            return Elem<T>::get(&tmp);
        };
        f32x4 vv = Elem<T>::get4(row + a.v_off + head * a.vp + v);
#pragma unroll
        for (int e = 0; e < 4; ++e) vv[e] = act(vv[e]);
        f32x4 o = {0, 0, 0, 0};
#pragma unroll
        for (int i = 0; i < ND; ++i)
            if (i < nd) {
                const float kk = act(Elem<T>::get(k + 32 * i)), qq = act(Elem<T>::get(q + 32 * i));
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    s[i][e] = fmaf(decay, s[i][e], kk * vv[e]);
                    o[e] = fmaf(s[i][e], qq, o[e]);
                }
            }
#pragma unroll
        for (int off = 8; off < 64; off <<= 1)
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] += __shfl_xor(o[e], off, kWave);
        if (lane < 8) *reinterpret_cast<f32x4*>(&red[t & 1][wave][lane * 4]) = o;
        __syncthreads();   // (two buffers: the next token's partial sums go to the other one)
        if (tid < 32) {
            const float x = (red[t & 1][0][tid] + red[t & 1][1][tid]) + (red[t & 1][2][tid] + red[t & 1][3][tid]);
            Elem<T>::put(static_cast<T*>(a.out) + (((int64_t)b * a.seq + t) * a.heads + head) * a.vp +
                             (int)blockIdx.x * 32 + tid, x);
        }
    }
#pragma unroll
    for (int i = 0; i < ND; ++i)
        if (i < nd) *reinterpret_cast<f32x4*>(state + (int64_t)(r + 32 * i) * a.vp) = s[i];
}

template <int DP, int VS>
void chunk_t(const LightningArgs& a, hipStream_t stream) {
    const dim3 grid((unsigned)a.nseg, (unsigned)((a.vp + VS - 1) / VS), (unsigned)(a.batch * a.heads));
    if (a.nseg > 1) {
        lightning_chunk_kernel<DP, VS, false><<<grid, 256, 0, stream>>>(a);
        const int64_t sz = (int64_t)a.dp * a.vp;
        lightning_scan_kernel<<<dim3((unsigned)((sz + 255) / 256), (unsigned)(a.batch * a.heads)), 256, 0, stream>>>(a);
    }
    lightning_chunk_kernel<DP, VS, true><<<grid, 256, 0, stream>>>(a);
}

template <int DP>
void chunk_d(const LightningArgs& a, hipStream_t stream) {
    if (a.vp <= 32) chunk_t<DP, 32>(a, stream);
    else chunk_t<DP, 64>(a, stream);
}

template <typename T>
void step_t(const LightningArgs& a, hipStream_t stream) {
    const dim3 grid((unsigned)(a.vp / 32), (unsigned)a.heads, (unsigned)a.batch);
    const int nd = a.dp / 32;
    if (nd <= 2) lightning_step_kernel<T, 2><<<grid, 256, 0, stream>>>(a);
    else if (nd <= 4) lightning_step_kernel<T, 4><<<grid, 256, 0, stream>>>(a);
    else if (nd <= 8) lightning_step_kernel<T, 8><<<grid, 256, 0, stream>>>(a);
    else lightning_step_kernel<T, 32><<<grid, 256, 0, stream>>>(a);
}

}  // namespace

bool lightning_chunk_supported(int dp, int vp) { return dp <= 256 && vp > 0; }

bool launch_lightning_chunk(const LightningArgs& a, hipStream_t stream) {
    if (!lightning_chunk_supported(a.dp, a.vp)) return false;
    if (a.dp <= 32) chunk_d<32>(a, stream);
    else if (a.dp <= 64) chunk_d<64>(a, stream);
    else if (a.dp <= 128) chunk_d<128>(a, stream);
    else chunk_d<256>(a, stream);
    return true;
}

bool lightning_step_supported(int dp, int vp) { return dp <= 1024 && vp > 0; }

void launch_lightning_step(const LightningArgs& a, int dtype, hipStream_t stream) {
    if (dtype) step_t<float>(a, stream);
    else step_t<uint16_t>(a, stream);
}

}  // namespace astrai_mix
