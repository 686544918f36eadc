// Grouped-query attention over cached keys and values, everything but the prompt kernel (mix_prefill.hip):
// RMS-normed and rotated queries and keys, soft-capped scores, a sink in the softmax denominator, a gate
// per output element -- each optional.
//
//   append   norms and rotates the queries in place and the new keys into the cache, copies the new values
//   rows     a few new tokens (bf16): the (token, head) rows of a group share every cached row; 16 of them
//            per workgroup, the context split over workgroups, its tiles of 32 keys over four waves that
//            work for themselves:
//              scores   v_mfma_f32_16x16x32_bf16 with keys as rows, operands straight from the cache;
//                       a lane holds keys 4 g .. and 16 + 4 g .. of one query, which is the next
//                       product's operand layout
//              values   the tile through the wave's own LDS, transposing reads; weights as two bf16 terms
//   merge    the splits, the sink and the gate
//   general  any size, bf16 or float, on the vector ALU: one workgroup per (token, head)
#include "mix_common.cuh"
#include "mix_launchers.h"

namespace astrai_mix {

namespace {

// `lanes` threads (8 columns each) per head row; rows of a token: queries, keys, values
template <typename T>
__global__ __launch_bounds__(256) void gqa_append_kernel(GqaAppendArgs a, GqaDims d, int lanes) {
    __shared__ __attribute__((aligned(16))) float ex[256 * 8];
    const int per_tok = d.heads + 2 * d.kv_heads;
    const int64_t item = (int64_t)blockIdx.x * (256 / lanes) + threadIdx.x / lanes;
    const int lane = threadIdx.x % lanes, col = lane * 8;
    bool live = item < a.tokens * per_tok;
    const int64_t t = live ? item / per_tok : 0, b = t / a.seq;
    const int r = live ? (int)(item - t * per_tok) : 0;
    const int64_t pos = a.positions[t - b * a.seq];
    live = live && pos >= 0 && pos < a.max_len && (!a.rot || pos < a.rot_rows);
    T* row = static_cast<T*>(a.proj) + t * a.ld;
    const int cs = d.dk + d.vp;
    T* cached = static_cast<T*>(a.cache) + (b * a.max_len + (live ? pos : 0)) * d.kv_heads * cs;
    const bool is_q = r < d.heads, is_k = !is_q && r < d.heads + d.kv_heads;
    const int h = is_q ? r : is_k ? r - d.heads : r - d.heads - d.kv_heads;
    const int width = is_q || is_k ? d.dk : d.vp;
    live = live && col < width;
    const T* src = row + (is_q ? h * d.dk : is_k ? a.k_off + h * d.dk : a.v_off + h * d.vp) + col;
    f32x4 x0 = {0, 0, 0, 0}, x1 = {0, 0, 0, 0};
    if (live) {
        x0 = Elem<T>::get4(src);
        x1 = Elem<T>::get4(src + 4);
    }
    const float* w = is_q ? a.q_norm : a.k_norm;
    float s = ((x0[0] * x0[0] + x0[1] * x0[1]) + (x0[2] * x0[2] + x0[3] * x0[3])) +
              ((x1[0] * x1[0] + x1[1] * x1[1]) + (x1[2] * x1[2] + x1[3] * x1[3]));
    for (int off = lanes / 2; off; off >>= 1) s += __shfl_xor(s, off, kWave);
    if ((is_q || is_k) && w && live) {
        const float f = 1.0f / sqrtf(s / (float)a.dim + a.eps);
        const f32x4 w0 = *reinterpret_cast<const f32x4*>(w + col), w1 = *reinterpret_cast<const f32x4*>(w + col + 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            x0[e] *= f * w0[e];
            x1[e] *= f * w1[e];
        }
    }
    float* mine = ex + threadIdx.x * 8;
    *reinterpret_cast<f32x4*>(mine) = x0;
    *reinterpret_cast<f32x4*>(mine + 4) = x1;
    __syncthreads();
    if (!live) return;
    if ((is_q || is_k) && a.rot && col < 2 * a.half) {
        const float* head = ex + (threadIdx.x - lane) * 8;
        const float2* rot = reinterpret_cast<const float2*>(a.rot) + pos * a.half;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const int i = col + e;
            if (i < 2 * a.half) {
                const bool first = i < a.half;
                const float2 c = rot[first ? i : i - a.half];
                const float own = head[i], other = head[first ? i + a.half : i - a.half];
                const float v = own * c.x + (first ? -other : other) * c.y;
                if (e < 4) x0[e] = v;
                else x1[e - 4] = v;
            }
        }
    }
    T* dst = is_q ? row + h * d.dk + col : cached + h * cs + (is_k ? 0 : d.dk) + col;
    Elem<T>::put4(dst, x0);
    Elem<T>::put4(dst + 4, x1);
}

// score in natural units
template <bool FAST>
__device__ __forceinline__ float score_of(float dot, const GqaDims& d) {
    const float s = dot * d.scale;
    if (d.softcap <= 0.0f) return s;
    return d.softcap * (FAST ? tanh_fast(s / d.softcap) : tanhf(s / d.softcap));
}

// NK key steps of 32 columns, NV value tiles of 16 columns
template <int NK, int NV>
__global__ __launch_bounds__(256) void gqa_partial_kernel(GqaRowsArgs a, GqaDims d) {
    constexpr int DV = NV * 16, kVRow = DV * 2 + 16, kAccRow = DV + 4;
    constexpr int CV = DV / 8, JV = 32 * CV / 64;      // 16-byte chunks of a value row, loads per lane
    constexpr int kTile = 32 * kVRow, kMerge = 16 * kAccRow * 4;
    __shared__ __attribute__((aligned(16))) uint8_t lds[4 * (kTile > kMerge ? kTile : kMerge)];
    __shared__ float ml[4][2][16];
    const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int split = (int)blockIdx.x % a.nsplit, rt = (int)blockIdx.x / a.nsplit, grp = blockIdx.y, b = blockIdx.z;
    const int rep = d.heads / d.kv_heads, rows = a.seq * rep;

    const int row = min(rt * 16 + c16, rows - 1), tok = row / rep, head = grp * rep + row - tok * rep;
    const int q_pos = (int)min(a.positions[tok], (int64_t)a.max_len - 1);
    const int q_lo = max(q_pos - d.window + 1, 0);
    // key range of the 16 rows: tokens in row order have rising positions
    const int kmax = (int)min(a.positions[min(rt * 16 + 15, rows - 1) / rep], (int64_t)a.max_len - 1);
    const int kmin = max((int)min(a.positions[rt * 16 / rep], (int64_t)a.max_len - 1) - d.window + 1, 0);
    const int tiles = (kmax - kmin + 32) >> 5, tps = (tiles + a.nsplit - 1) / a.nsplit;
    const int t0 = split * tps, t1 = min(t0 + tps, tiles);

    u32x4 qf[NK];
    {
        const uint16_t* q = static_cast<const uint16_t*>(a.proj) + ((int64_t)b * a.seq + tok) * a.ld + head * d.dk + 8 * g;
#pragma unroll
        for (int i = 0; i < NK; ++i) qf[i] = i * 32 < d.dk ? *reinterpret_cast<const u32x4*>(q + i * 32) : u32x4{0, 0, 0, 0};
    }
    // keys past kmax read as zeros, columns past the real ones too
    const uint32_t ldc = (uint32_t)(d.kv_heads * (d.dk + d.vp)) * 2, cs = (uint32_t)(d.dk + d.vp) * 2;   // bytes
    const __amdgpu_buffer_rsrc_t rc = w8a8::make_rsrc(
        static_cast<const uint8_t*>(a.cache) + (int64_t)b * a.max_len * ldc + grp * cs, (uint32_t)kmax * ldc + cs);
    u32x4 kf[2][NK], vf[JV];
    auto fetch = [&](int t) {
        const uint32_t key = (uint32_t)(kmin + t * 32);
        const bool in = t < t1;
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int i = 0; i < NK; ++i)
                kf[u][i] = w8a8::buf_load16(rc, in && i * 32 < d.dk ? (key + u * 16 + c16) * ldc + i * 64 + 16 * g
                                                                    : w8a8::kOutOfRange, 0);
#pragma unroll
        for (int i = 0; i < JV; ++i) {
            const int r = i * (64 / CV) + lane / CV, c = lane % CV;
            // (a row past kmax starts past the buffer's end: kmax's own row ends it)
            vf[i] = w8a8::buf_load16(rc, in && c * 8 < d.vp ? (key + r) * ldc + d.dk * 2 + c * 16 : w8a8::kOutOfRange, 0);
        }
    };
    uint8_t* const vt = lds + wave * kTile;
    f32x4 acc[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) acc[i] = f32x4{0, 0, 0, 0};
    float m = kNegBig, l = 0.0f;   // log2 units; l: this lane's keys only
    fetch(t0 + wave);
    for (int t = t0 + wave; t < t1; t += 4) {
        f32x4 s[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}};
#pragma unroll
        for (int i = 0; i < NK; ++i) {
            s[0] = mfma16(kf[0][i], qf[i], s[0]);
            s[1] = mfma16(kf[1][i], qf[i], s[1]);
        }
#pragma unroll
        for (int i = 0; i < JV; ++i)
            *reinterpret_cast<u32x4*>(vt + (i * (64 / CV) + lane / CV) * kVRow + (lane % CV) * 16) = vf[i];
        fetch(t + 4);
        float tm = kNegBig;
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int key = kmin + t * 32 + u * 16 + 4 * g + e;
                s[u][e] = (key <= q_pos && key >= q_lo) ? score_of<true>(s[u][e], d) * kLog2e : kNegBig;
                tm = fmaxf(tm, s[u][e]);
            }
        tm = fmaxf(tm, __shfl_xor(tm, 16, kWave));
        tm = fmaxf(tm, __shfl_xor(tm, 32, kWave));
        const float m_new = fmaxf(m, tm), alpha = __builtin_amdgcn_exp2f(m - m_new);
        m = m_new;
        l *= alpha;
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                s[u][e] = s[u][e] > 0.5f * kNegBig ? __builtin_amdgcn_exp2f(s[u][e] - m_new) : 0.0f;
                l += s[u][e];
            }
        u32x4 hi, lo;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            uint32_t h0, l0, h1, l1;
            split2(s[u][0], s[u][1], h0, l0);
            split2(s[u][2], s[u][3], h1, l1);
            hi[2 * u] = h0;
            hi[2 * u + 1] = h1;
            lo[2 * u] = l0;
            lo[2 * u + 1] = l1;
        }
        __builtin_amdgcn_wave_barrier();   // the tile in LDS is this wave's own
        const uint8_t* src = vt + (4 * g + (c16 >> 2)) * kVRow + (c16 & 3) * 8;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const u32x4 v = join(lds_read_tr(src + i * 32), lds_read_tr(src + i * 32 + 16 * kVRow));
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[i][e] *= alpha;
            acc[i] = mfma16(v, hi, acc[i]);
            acc[i] = mfma16(v, lo, acc[i]);
        }
        __builtin_amdgcn_wave_barrier();
    }
    l += __shfl_xor(l, 16, kWave);
    l += __shfl_xor(l, 32, kWave);
    __syncthreads();
    // the four waves' parts of each query: [wave][query][DV]
    float* const part = reinterpret_cast<float*>(lds);
#pragma unroll
    for (int i = 0; i < NV; ++i)
        *reinterpret_cast<f32x4*>(part + (wave * 16 + c16) * kAccRow + 16 * i + 4 * g) = acc[i];
    if (g == 0) {
        ml[wave][0][c16] = m;
        ml[wave][1][c16] = l;
    }
    __syncthreads();
    // workspace per (row, split): vp values, then maximum and sum
    for (int i = tid; i < 16 * (DV / 4); i += 256) {
        const int q = i / (DV / 4), col = i % (DV / 4) * 4;
        if (rt * 16 + q >= rows || col >= d.vp) continue;
        const float m4[4] = {ml[0][0][q], ml[1][0][q], ml[2][0][q], ml[3][0][q]};
        const float big = fmaxf(fmaxf(m4[0], m4[1]), fmaxf(m4[2], m4[3]));
        f32x4 o = {0, 0, 0, 0};
        float sum = 0.0f;
#pragma unroll
        for (int w = 0; w < 4; ++w) {
            const float f = __builtin_amdgcn_exp2f(m4[w] - big);
            const f32x4 v = *reinterpret_cast<const f32x4*>(part + (w * 16 + q) * kAccRow + col);
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] = fmaf(f, v[e], o[e]);
            sum = fmaf(f, ml[w][1][q], sum);
        }
        float* ws = a.ws + ((((int64_t)b * d.kv_heads + grp) * rows + rt * 16 + q) * a.nsplit + split) * (d.vp + 4);
        *reinterpret_cast<f32x4*>(ws + col) = o;
        if (col == 0) {
            ws[d.vp] = big;
            ws[d.vp + 1] = sum;
        }
    }
}

// one workgroup of 64 per (sequence, group, row)
__global__ __launch_bounds__(64) void gqa_merge_kernel(GqaRowsArgs a, GqaDims d) {
    __shared__ float wt[kMaxSplit];
    const int lane = threadIdx.x, rep = d.heads / d.kv_heads, rows = a.seq * rep;
    const int row = blockIdx.x, grp = blockIdx.y, b = blockIdx.z;
    const int tok = row / rep, head = grp * rep + row - tok * rep;
    const int ldw = d.vp + 4;
    const float* w = a.ws + (((int64_t)b * d.kv_heads + grp) * rows + row) * a.nsplit * ldw;
    // (a split without a key has maximum kNegBig and sum 0)
    const f32x2 ml = lane < a.nsplit ? *reinterpret_cast<const f32x2*>(w + (int64_t)lane * ldw + d.vp) : f32x2{kNegBig, 0.0f};
    const float big = fmaxf(w8a8::wave_max(ml[0]), d.sink ? 0.0f : kNegBig);
    const float e = __builtin_amdgcn_exp2f(ml[0] - big);
    float sum = wave_sum(ml[1] * e);
    if (d.sink) sum += __builtin_amdgcn_exp2f(-big);
    if (lane < a.nsplit) wt[lane] = sum > 0.0f ? e / sum : 0.0f;
    __syncthreads();
    const int64_t t = (int64_t)b * a.seq + tok;
    for (int c = lane * 4; c < d.vp; c += 256) {
        f32x4 o = {0, 0, 0, 0};
#pragma unroll 4
        for (int s = 0; s < a.nsplit; ++s) {
            const f32x4 v = *reinterpret_cast<const f32x4*>(w + (int64_t)s * ldw + c);
            const float f = wt[s];
#pragma unroll
            for (int j = 0; j < 4; ++j) o[j] = fmaf(f, v[j], o[j]);
        }
        if (a.g_off >= 0) {
            const f32x4 z = Elem<uint16_t>::get4(static_cast<const uint16_t*>(a.proj) + t * a.ld + a.g_off + head * d.vp + c);
#pragma unroll
            for (int j = 0; j < 4; ++j) o[j] *= sigmoid_fast(z[j]);
        }
        Elem<uint16_t>::put4(static_cast<uint16_t*>(a.out) + (t * d.heads + head) * d.vp + c, o);
    }
}

constexpr int kGenCols = 1024;   // key or value columns a workgroup can hold

template <typename T>
__global__ __launch_bounds__(256) void gqa_general_kernel(GqaRowsArgs a, GqaDims d) {
    __shared__ float qs[kGenCols];
    __shared__ float ps[256];
    __shared__ float slots[kRowThreads / kWave];
    const int tid = threadIdx.x, h = blockIdx.y, grp = h / (d.heads / d.kv_heads);
    const int64_t t = blockIdx.x, b = t / a.seq;
    const int pos = (int)min(a.positions[t - b * a.seq], (int64_t)a.max_len - 1);
    for (int c = tid; c < d.dk; c += 256) qs[c] = Elem<T>::get(static_cast<const T*>(a.proj) + t * a.ld + h * d.dk + c);
    __syncthreads();
    const int cs = d.dk + d.vp, ldc = d.kv_heads * cs;
    const T* cache = static_cast<const T*>(a.cache) + b * a.max_len * ldc + grp * cs;
    float acc[kGenCols / 256];
#pragma unroll
    for (int i = 0; i < kGenCols / 256; ++i) acc[i] = 0.0f;
    float m = d.sink ? 0.0f : kNegBig, l = d.sink ? 1.0f : 0.0f;
    for (int k0 = max(pos - d.window + 1, 0); k0 <= pos; k0 += 256) {
        const int n = min(256, pos + 1 - k0);
        float s = kNegBig;
        if (tid < n) {
            const T* row = cache + (int64_t)(k0 + tid) * ldc;
            float x = 0.0f;
            for (int e = 0; e < d.dk; e += 4) {
                const f32x4 v = Elem<T>::get4(row + e);
#pragma unroll
                for (int j = 0; j < 4; ++j) x = fmaf(v[j], qs[e + j], x);
            }
            s = score_of<false>(x, d);
        }
        const float m_new = fmaxf(m, w8a8::block_max(s, slots));
        const float alpha = expf(m - m_new);
        const float p = tid < n ? expf(s - m_new) : 0.0f;
        ps[tid] = p;
        l = l * alpha + block_sum(p, slots);   // (its barriers also publish ps)
        m = m_new;
#pragma unroll
        for (int i = 0; i < kGenCols / 256; ++i) {
            const int c = tid + i * 256;
            if (c < d.vp) {
                float o = acc[i] * alpha;
                for (int j = 0; j < n; ++j) o = fmaf(ps[j], Elem<T>::get(cache + (int64_t)(k0 + j) * ldc + d.dk + c), o);
                acc[i] = o;
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < kGenCols / 256; ++i) {
        const int c = tid + i * 256;
        if (c < d.vp) {
            float o = acc[i] / l;
            if (a.g_off >= 0) o *= sigmoid(Elem<T>::get(static_cast<const T*>(a.proj) + t * a.ld + a.g_off + h * d.vp + c));
            Elem<T>::put(static_cast<T*>(a.out) + (t * d.heads + h) * d.vp + c, o);
        }
    }
}

template <int NK, int NV>
void partial_t(const GqaRowsArgs& a, const GqaDims& d, hipStream_t stream) {
    const int rows = a.seq * (d.heads / d.kv_heads);
    const dim3 grid((unsigned)a.nsplit * (unsigned)((rows + 15) / 16), (unsigned)d.kv_heads, (unsigned)a.batch);
    gqa_partial_kernel<NK, NV><<<grid, 256, 0, stream>>>(a, d);
}

template <int NK>
void partial_v(const GqaRowsArgs& a, const GqaDims& d, hipStream_t stream) {
    if (d.vp <= 64) partial_t<NK, 4>(a, d, stream);
    else partial_t<NK, 8>(a, d, stream);
}

}  // namespace

void launch_gqa_append(const GqaAppendArgs& a, const GqaDims& d, int dtype, hipStream_t stream) {
    int lanes = 4;
    while (lanes < 64 && lanes * 8 < (d.dk > d.vp ? d.dk : d.vp)) lanes *= 2;
    const int64_t items = a.tokens * (d.heads + 2 * d.kv_heads), per = 256 / lanes;
    const dim3 grid((unsigned)((items + per - 1) / per));
    if (dtype) gqa_append_kernel<float><<<grid, 256, 0, stream>>>(a, d, lanes);
    else gqa_append_kernel<uint16_t><<<grid, 256, 0, stream>>>(a, d, lanes);
}

bool gqa_rows_mfma_supported(const GqaDims& d) { return d.dk <= 256 && d.vp <= 128; }

int64_t gqa_rows_workspace_floats(const GqaDims& d, int64_t tokens, int nsplit) {
    return tokens * d.heads * nsplit * (d.vp + 4);
}

void launch_gqa_rows_mfma(const GqaRowsArgs& a, const GqaDims& d, hipStream_t stream) {
    if (d.dk <= 64) partial_v<2>(a, d, stream);
    else if (d.dk <= 128) partial_v<4>(a, d, stream);
    else partial_v<8>(a, d, stream);
    const int rows = a.seq * (d.heads / d.kv_heads);
    gqa_merge_kernel<<<dim3((unsigned)rows, (unsigned)d.kv_heads, (unsigned)a.batch), 64, 0, stream>>>(a, d);
}

bool gqa_rows_general_supported(const GqaDims& d) { return d.dk <= kGenCols && d.vp <= kGenCols; }

void launch_gqa_rows_general(const GqaRowsArgs& a, const GqaDims& d, int dtype, hipStream_t stream) {
    const dim3 grid((unsigned)((int64_t)a.batch * a.seq), (unsigned)d.heads);
    if (dtype) gqa_general_kernel<float><<<grid, 256, 0, stream>>>(a, d);
    else gqa_general_kernel<uint16_t><<<grid, 256, 0, stream>>>(a, d);
}

}  // namespace astrai_mix
