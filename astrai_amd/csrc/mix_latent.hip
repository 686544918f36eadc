// Latent attention, everything but the prompt kernel: per-head keys and values are projections
// W_uk c, W_uv c of a cached latent c, plus one rotated key part shared by all heads.
//
//   latent_append   rotates the queries' rotated parts in place, norms the new latents, rotates
//                   the new key parts and writes both into the cache; for the rows path it also absorbs
//                   W_uk into the queries
//   rows path       a few new tokens against the cache without ever forming keys or values:
//                   q_u . (W_uk c) = (W_uk^T q_u) . c, and the output is W_uv (sum p c). With the
//                   projection absorbed into the query, all heads of a token share one key/value
//                   row per position, so the cache is read once per 16 (token, head) rows.
//     absorb        q_abs[t, h] = W_uk[h]^T q_u[t, h]            (MFMA, weight-streaming)
//     partial       split-context attention in the latent space  (MFMA)
//     merge         splits of a row into one attended latent
//     expand        W_uv[h] applied, output gate                 (MFMA, weight-streaming)
//   general path  the same steps on the vector ALU for any size and for float, one kernel
#include "mix_common.cuh"
#include "mix_launchers.h"

namespace astrai_mix {

namespace {

// ---- append: N threads (a wave or a workgroup) per token --------------------------------------------
template <typename T, int N>
__device__ __forceinline__ void append_token(const LatentAppendArgs& a, const LatentDims& d, int64_t t, int lane,
                                             float* slots) {
    const int64_t b = t / a.seq;
    const int64_t pos = a.positions[t - b * a.seq];
    if (pos < 0 || pos >= a.max_len || pos >= a.rot_rows) return;   // (the same for the token's N threads)
    T* row = static_cast<T*>(a.proj) + t * a.ld;
    const float2* rot = reinterpret_cast<const float2*>(a.rot) + pos * a.half;
    const int qs = d.dn + d.dr;
    for (int i = lane; i < d.heads * a.half; i += N) {
        const int h = i / a.half, p = i - h * a.half;
        T* u = row + h * qs + d.dn + p;
        const float2 cs = rot[p];
        const float x = Elem<T>::get(u), y = Elem<T>::get(u + a.half);
        Elem<T>::put(u, x * cs.x - y * cs.y);
        Elem<T>::put(u + a.half, y * cs.x + x * cs.y);
    }
    if (a.dkv_off < 0) return;
    const T* src = row + a.dkv_off;
    T* dst = static_cast<T*>(a.cache) + (b * a.max_len + pos) * (d.rp + d.dr);
    float s = 0.0f;
    for (int c = lane * 4; c < d.rp; c += 4 * N) {
        const f32x4 v = Elem<T>::get4(src + c);
        s += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
    }
    const float r = 1.0f / sqrtf((N == 64 ? wave_sum(s) : block_sum(s, slots)) / (float)a.kv_rank + a.eps);
    for (int c = lane * 4; c < d.rp; c += 4 * N) {
        f32x4 v = Elem<T>::get4(src + c);
        const f32x4 w = *reinterpret_cast<const f32x4*>(a.norm_w + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = v[e] * r * w[e];
        Elem<T>::put4(dst + c, v);
    }
    src += d.rp;
    dst += d.rp;
    for (int p = lane; p < a.half; p += N) {
        const float2 cs = rot[p];
        const float x = Elem<T>::get(src + p), y = Elem<T>::get(src + p + a.half);
        Elem<T>::put(dst + p, x * cs.x - y * cs.y);
        Elem<T>::put(dst + p + a.half, y * cs.x + x * cs.y);
    }
    for (int p = 2 * a.half + lane; p < d.dr; p += N) dst[p] = src[p];
}

// a wave per token (prompts)
template <typename T>
__global__ __launch_bounds__(256) void latent_append_kernel(LatentAppendArgs a, LatentDims d) {
    const int64_t t = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t < a.tokens) append_token<T, 64>(a, d, t, threadIdx.x & 63, nullptr);
}

// A few tokens: the first a.tokens workgroups append one each. The others absorb W_uk into the queries,
//   q_abs[t, h, r] = sum_d q[t, h, d] w_uk_t[h, r, d]
// over the unrotated columns, which the append leaves alone: one wave per (16 latent columns, head, 16
// tokens). Weight rows are the MFMA's rows and tokens its columns, so a lane ends up with four consecutive
// columns of one token; both operands come straight from memory, 16 bytes a lane.
template <typename T>
__global__ __launch_bounds__(256) void latent_append_few_kernel(LatentAppendArgs a, LatentDims d) {
    __shared__ float slots[kRowThreads / kWave];
    if ((int64_t)blockIdx.x < a.tokens) {
        append_token<T, 256>(a, d, blockIdx.x, threadIdx.x, slots);
        return;
    }
    if constexpr (sizeof(T) == 2) {
        const int nb = (d.rp + 63) / 64;
        int item = (int)((int64_t)blockIdx.x - a.tokens);
        const int lane = threadIdx.x & 63, c16 = lane & 15, g = lane >> 4;
        const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
        const int r0 = ((item % nb) * 4 + wave) * 16;
        item /= nb;
        const int h = item % d.heads;
        const int64_t t = (int64_t)(item / d.heads) * 16 + c16;
        if (r0 >= d.rp) return;
        const int64_t tl = min(t, a.tokens - 1);   // (a row past the end repeats the last one and is not stored)
        const uint16_t* x = static_cast<const uint16_t*>(a.proj) + tl * a.ld + h * (d.dn + d.dr) + 8 * g;
        const uint16_t* w = static_cast<const uint16_t*>(a.w_uk_t) + ((int64_t)h * d.rp + r0 + c16) * d.dn + 8 * g;
        f32x4 acc = {0, 0, 0, 0};
#pragma unroll 4
        for (int k = 0; k < d.dn; k += 32)
            acc = mfma16(*reinterpret_cast<const u32x4*>(w + k), *reinterpret_cast<const u32x4*>(x + k), acc);
        if (t < a.tokens)
            Elem<uint16_t>::put4(static_cast<uint16_t*>(a.q_abs) + (t * d.heads + h) * d.rp + r0 + 4 * g, acc);
    }
}

// ---- split-context attention over the latent rows (bf16) -------------------------------------------
// Rows are (token, head) pairs of one sequence, token-major; a workgroup takes 16 of them and one
// split of the keys, in tiles of 32. Four waves:
//   scores   wave (kh, ch) multiplies keys 16 kh .. of the tile with latent steps RH ch .. RH ch + RH - 1 (of
//            32 columns) and rotated step ch; its key operand comes straight from the cache, and the
//            latent registers are written to LDS for the value product. The halves meet in LDS.
//   softmax  fp32, every wave for itself: lane (query c16, group g) holds keys 8g .. 8g+7, which is
//            the value product's operand layout. Probabilities go in as two bf16 terms.
//   values   wave w accumulates latent columns 16 (w + 4 i) .., the transposed operand out of LDS.
// The LDS tiles alternate between two buffers: one barrier per tile; key operands are requested two
// tiles ahead. Nothing in a tile branches: with fewer latent columns than 64 RH, the steps past them
// meet zero query operands and fill LDS columns that are never stored.
template <int RH>
__global__ __launch_bounds__(256, RH <= 8 ? 2 : 1) void latent_partial_kernel(LatentRowsArgs a, LatentDims d) {
    constexpr int kScRow = 36;                       // floats per query row of scores (32 + padding)
    constexpr int kVRow = RH * 128 + 32;             // bytes per latent row in LDS
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    const int lane = threadIdx.x & 63, c16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int kh = wave & 1, ch = wave >> 1;
    const int split = (int)blockIdx.x % a.nsplit, rt = (int)blockIdx.x / a.nsplit, b = blockIdx.y;
    const int rows = a.seq * d.heads;
    float* sc = reinterpret_cast<float*>(lds + 2 * 32 * kVRow);

    const int row = rt * 16 + c16;
    const bool live = row < rows;
    const int tok = min(row, rows - 1) / d.heads, head = min(row, rows - 1) - tok * d.heads;
    const int q_pos = (int)min(a.positions[tok], (int64_t)a.max_len - 1);
    const int q_lo = max(q_pos - d.window + 1, 0);
    // key range of the 16 rows: tokens in row order have rising positions
    const int tok0 = rt * 16 / d.heads, tok1 = min(rt * 16 + 15, rows - 1) / d.heads;
    const int kmax = (int)min(a.positions[tok1], (int64_t)a.max_len - 1);
    const int kmin = max((int)min(a.positions[tok0], (int64_t)a.max_len - 1) - d.window + 1, 0);
    const int tiles = (kmax - kmin + 32) >> 5;
    const int tps = (tiles + a.nsplit - 1) / a.nsplit;
    const int t0 = split * tps, t1 = min(t0 + tps, tiles);

    const u32x4 zero = {0, 0, 0, 0};
    u32x4 qf[RH + 1];   // query operand of this wave's steps; the rotated one last
    {
        const int64_t t = (int64_t)b * a.seq + tok;
        const uint16_t* qa = static_cast<const uint16_t*>(a.q_abs) + (t * d.heads + head) * d.rp;
        const uint16_t* qr = static_cast<const uint16_t*>(a.proj) + t * a.ld + head * (d.dn + d.dr) + d.dn;
#pragma unroll
        for (int i = 0; i < RH; ++i) {
            const int e = (ch * RH + i) * 32 + 8 * g;
            qf[i] = (e < d.rp && live) ? *reinterpret_cast<const u32x4*>(qa + e) : zero;
        }
        qf[RH] = (ch * 32 < d.dr && live) ? *reinterpret_cast<const u32x4*>(qr + ch * 32 + 8 * g) : zero;
    }
    // keys past kmax read as zeros
    const uint32_t ldc = (uint32_t)(d.rp + d.dr) * 2;   // bytes
    const __amdgpu_buffer_rsrc_t rc = w8a8::make_rsrc(
        static_cast<const uint8_t*>(a.cache) + (int64_t)b * a.max_len * ldc, (uint32_t)(kmax + 1) * ldc);
    const uint32_t lane_c = (uint32_t)(ch * RH * 64 + 16 * g), lane_r = (uint32_t)(d.rp * 2 + ch * 64 + 16 * g);
    u32x4 ka[RH + 1], kb[RH + 1];   // key operands of two tiles in flight
    auto fetch = [&](int t, u32x4 (&kf)[RH + 1]) {
        const uint32_t off = t < t1 ? (uint32_t)(kmin + t * 32 + kh * 16 + c16) * ldc : w8a8::kOutOfRange;
#pragma unroll
        for (int i = 0; i < RH; ++i) kf[i] = w8a8::buf_load16(rc, off + lane_c + i * 64, 0);
        kf[RH] = w8a8::buf_load16(rc, ch * 32 < d.dr ? off + lane_r : w8a8::kOutOfRange, 0);
    };
    fetch(t0, ka);
    fetch(t0 + 1, kb);

    f32x4 acc[RH];
#pragma unroll
    for (int i = 0; i < RH; ++i) acc[i] = f32x4{0, 0, 0, 0};
    float m = kNegBig, l = 0.0f;   // l: this lane's keys only
    const float c = d.scale * kLog2e;
    auto tile = [&](int t, int buf, u32x4 (&kf)[RH + 1]) {
        uint8_t* v = lds + buf * 32 * kVRow;
        float* s = sc + buf * 2 * 16 * kScRow;
        f32x4 part[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}};
#pragma unroll
        for (int i = 0; i <= RH; ++i) {
            part[i & 1] = mfma16(kf[i], qf[i], part[i & 1]);
            if (i < RH)
                *reinterpret_cast<u32x4*>(v + (kh * 16 + c16) * kVRow + (ch * RH + i) * 64 + 16 * g) = kf[i];
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) part[0][e] += part[1][e];
        *reinterpret_cast<f32x4*>(s + (ch * 16 + c16) * kScRow + kh * 16 + 4 * g) = part[0];
        fetch(t + 2, kf);
        __syncthreads();
        float p[8], tm = kNegBig;
        const float* s0 = s + c16 * kScRow + 8 * g;
        const float* s1 = s0 + 16 * kScRow;
#pragma unroll
        for (int e = 0; e < 8; e += 4) {
            const f32x4 x = *reinterpret_cast<const f32x4*>(s0 + e), y = *reinterpret_cast<const f32x4*>(s1 + e);
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int key = kmin + t * 32 + 8 * g + e + j;
                p[e + j] = (key <= q_pos && key >= q_lo) ? (x[j] + y[j]) * c : kNegBig;
                tm = fmaxf(tm, p[e + j]);
            }
        }
        tm = fmaxf(tm, __shfl_xor(tm, 16, kWave));
        tm = fmaxf(tm, __shfl_xor(tm, 32, kWave));
        const float m_new = fmaxf(m, tm);
        const float alpha = __builtin_amdgcn_exp2f(m - m_new);
        m = m_new;
        l *= alpha;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            p[e] = p[e] > 0.5f * kNegBig ? __builtin_amdgcn_exp2f(p[e] - m_new) : 0.0f;
            l += p[e];
        }
        u32x4 hi, lo;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            uint32_t h2, l2;
            split2(p[2 * e], p[2 * e + 1], h2, l2);
            hi[e] = h2;
            lo[e] = l2;
        }
        // transposed latent operand: 16 columns x 32 keys, lane group g takes keys 8g .. 8g+7
        const uint8_t* src = v + (8 * g + (c16 >> 2)) * kVRow + (c16 & 3) * 8 + wave * 32;
#pragma unroll
        for (int i = 0; i < RH; ++i) {
            const u32x4 vf = join(lds_read_tr(src + i * 128), lds_read_tr(src + i * 128 + 4 * kVRow));
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[i][e] *= alpha;
            acc[i] = mfma16(vf, hi, acc[i]);
            acc[i] = mfma16(vf, lo, acc[i]);
        }
    };
    for (int t = t0; t < t1; t += 2) {
        tile(t, 0, ka);
        if (t + 1 < t1) tile(t + 1, 1, kb);
    }
    l += __shfl_xor(l, 16, kWave);
    l += __shfl_xor(l, 32, kWave);
    if (!live) return;
    // workspace per (row, split): rp values, then maximum and sum
    float* w = a.ws + (((int64_t)b * rows + row) * a.nsplit + split) * (d.rp + 4);
#pragma unroll
    for (int i = 0; i < RH; ++i) {
        const int col = (wave + 4 * i) * 16;
        if (col < d.rp) *reinterpret_cast<f32x4*>(w + col + 4 * g) = acc[i];
    }
    if (wave == 0 && g == 0) {
        w[d.rp] = m;
        w[d.rp + 1] = l;
    }
}

// ---- merge the splits of a (token, head) row (bf16): one workgroup of 128 per row -------------------
__global__ __launch_bounds__(128) void latent_merge_kernel(LatentRowsArgs a, LatentDims d) {
    __shared__ float wt[kMaxSplit];
    const int64_t row = blockIdx.x;
    const int tid = threadIdx.x, lane = tid & 63;
    const int ldw = d.rp + 4;
    const float* w = a.ws + row * a.nsplit * ldw;
    // (a split without a key has maximum kNegBig and sum 0)
    const f32x2 ml = lane < a.nsplit ? *reinterpret_cast<const f32x2*>(w + (int64_t)lane * ldw + d.rp) : f32x2{kNegBig, 0.0f};
    const float big = w8a8::wave_max(ml[0]);
    const float e = __builtin_amdgcn_exp2f(ml[0] - big);
    const float sum = wave_sum(ml[1] * e);
    if (tid < a.nsplit) wt[tid] = sum > 0.0f ? e / sum : 0.0f;
    __syncthreads();
    for (int r = tid * 4; r < d.rp; r += 512) {
        f32x4 o = {0, 0, 0, 0};
#pragma unroll 4
        for (int s = 0; s < a.nsplit; ++s) {
            const f32x4 v = *reinterpret_cast<const f32x4*>(w + (int64_t)s * ldw + r);
            const float f = wt[s];
#pragma unroll
            for (int j = 0; j < 4; ++j) o[j] += f * v[j];
        }
        Elem<uint16_t>::put4(static_cast<uint16_t*>(a.o_lat) + row * d.rp + r, o);
    }
}

// ---- expand (bf16): out[t, h, v] = sigmoid(gate) sum_r o_lat[t, h, r] W_uv[h, v, r] --------------------
// One workgroup per (16 value columns, head, 16 tokens), the waves sharing out the latent columns, so
// that a wave's operands are one round of loads. Layouts as in absorb.
__global__ __launch_bounds__(256) void latent_expand_kernel(LatentRowsArgs a, LatentDims d) {
    __shared__ f32x4 part[3][64];
    const int lane = threadIdx.x & 63, c16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int v0 = (int)blockIdx.x * 16, h = blockIdx.y;
    const int64_t tokens = (int64_t)a.batch * a.seq;
    const int64_t t = (int64_t)blockIdx.z * 16 + c16;
    const int64_t tl = min(t, tokens - 1);
    const float z = Elem<uint16_t>::get(static_cast<const uint16_t*>(a.proj) + tl * a.ld + a.g_off + h);
    const uint16_t* x = static_cast<const uint16_t*>(a.o_lat) + (tl * d.heads + h) * d.rp + 8 * g;
    const uint16_t* w = static_cast<const uint16_t*>(a.w_ukv) + ((int64_t)h * (d.dn + d.vp) + d.dn + v0 + c16) * d.rp + 8 * g;
    f32x4 acc = {0, 0, 0, 0};
#pragma unroll 4
    for (int k = wave * 32; k < d.rp; k += 128)
        acc = mfma16(*reinterpret_cast<const u32x4*>(w + k), *reinterpret_cast<const u32x4*>(x + k), acc);
    if (wave) part[wave - 1][lane] = acc;
    __syncthreads();
    if (wave || t >= tokens) return;
    const float gate = sigmoid(z);
#pragma unroll
    for (int e = 0; e < 4; ++e)
        acc[e] = ((acc[e] + part[0][lane][e]) + (part[1][lane][e] + part[2][lane][e])) * gate;
    Elem<uint16_t>::put4(static_cast<uint16_t*>(a.out) + (t * d.heads + h) * d.vp + v0 + 4 * g, acc);
}

// ---- general path: any size, bf16 or float, one workgroup per (head, token) ---------------------------
constexpr int kGenRank = 2048;   // latent columns a workgroup can hold (8 per thread)
constexpr int kGenDims = 512;    // query dimensions of either kind

template <typename T>
__global__ __launch_bounds__(256) void latent_general_kernel(LatentRowsArgs a, LatentDims d) {
    __shared__ float qs[kGenRank + kGenDims];
    __shared__ float ps[256];
    __shared__ float slots[kRowThreads / kWave];
    const int tid = threadIdx.x, h = blockIdx.y;
    const int64_t t = blockIdx.x;
    const int64_t b = t / a.seq;
    const int pos = (int)min(a.positions[t - b * a.seq], (int64_t)a.max_len - 1);
    const T* q = static_cast<const T*>(a.proj) + t * a.ld + h * (d.dn + d.dr);
    const T* wk = static_cast<const T*>(a.w_ukv) + (int64_t)h * (d.dn + d.vp) * d.rp;
    const int ldc = d.rp + d.dr;
    // absorb; rounded to the activation type, as the matrix-core path hands it on
    for (int r = tid; r < d.rp; r += 256) {
        float s = 0.0f;
        for (int k = 0; k < d.dn; ++k) s = fmaf(Elem<T>::get(q + k), Elem<T>::get(wk + (int64_t)k * d.rp + r), s);
        T tmp;
        Elem<T>::put(&tmp, s);
        qs[r] = Elem<T>::get(&tmp);
    }
    for (int r = tid; r < d.dr; r += 256) qs[d.rp + r] = Elem<T>::get(q + d.dn + r);
    __syncthreads();
    const T* cache = static_cast<const T*>(a.cache) + b * a.max_len * ldc;
    float acc[kGenRank / 256];
#pragma unroll
    for (int i = 0; i < kGenRank / 256; ++i) acc[i] = 0.0f;
    float m = kNegBig, l = 0.0f;
    for (int k0 = max(pos - d.window + 1, 0); k0 <= pos; k0 += 256) {
        const int n = min(256, pos + 1 - k0);
        float s = kNegBig;
        if (tid < n) {
            const T* row = cache + (int64_t)(k0 + tid) * ldc;
            float x = 0.0f;
            for (int e = 0; e < ldc; e += 4) {
                const f32x4 v = Elem<T>::get4(row + e);
#pragma unroll
                for (int j = 0; j < 4; ++j) x = fmaf(v[j], qs[e + j], x);
            }
            s = x * d.scale;
        }
        const float m_new = fmaxf(m, w8a8::block_max(s, slots));
        const float alpha = expf(m - m_new);
        const float p = tid < n ? expf(s - m_new) : 0.0f;
        ps[tid] = p;
        l = l * alpha + block_sum(p, slots);   // (its barriers also publish ps)
        m = m_new;
#pragma unroll
        for (int i = 0; i < kGenRank / 256; ++i) {
            const int r = tid + i * 256;
            if (r < d.rp) {
                float o = acc[i] * alpha;
                for (int j = 0; j < n; ++j) o = fmaf(ps[j], Elem<T>::get(cache + (int64_t)(k0 + j) * ldc + r), o);
                acc[i] = o;
            }
        }
        __syncthreads();
    }
    const float inv = 1.0f / l;
    for (int i = 0; i < kGenRank / 256; ++i) {
        const int r = tid + i * 256;
        if (r < d.rp) {
            T tmp;
            Elem<T>::put(&tmp, acc[i] * inv);
            qs[r] = Elem<T>::get(&tmp);
        }
    }
    __syncthreads();
    const float gate = sigmoid(Elem<T>::get(static_cast<const T*>(a.proj) + t * a.ld + a.g_off + h));
    for (int v = tid; v < d.vp; v += 256) {
        const T* wv = wk + (int64_t)(d.dn + v) * d.rp;
        float s = 0.0f;
        for (int r = 0; r < d.rp; r += 4) {
            const f32x4 w = Elem<T>::get4(wv + r);
#pragma unroll
            for (int j = 0; j < 4; ++j) s = fmaf(w[j], qs[r + j], s);
        }
        Elem<T>::put(static_cast<T*>(a.out) + (t * d.heads + h) * d.vp + v, s * gate);
    }
}

template <int RH>
void partial_t(const LatentRowsArgs& a, const LatentDims& d, hipStream_t stream) {
    constexpr int shared = 2 * 32 * (RH * 128 + 32) + 2 * 2 * 16 * 36 * (int)sizeof(float);
    static const hipError_t once = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_partial_kernel<RH>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, shared);
    (void)once;
    const int rows = a.seq * d.heads;
    const dim3 grid((unsigned)a.nsplit * (unsigned)((rows + 15) / 16), (unsigned)a.batch);
    latent_partial_kernel<RH><<<grid, 256, shared, stream>>>(a, d);
}

}  // namespace

void launch_latent_append(const LatentAppendArgs& a, const LatentDims& d, int dtype, hipStream_t stream) {
    if (a.q_abs || a.tokens <= 1024) {
        const int64_t absorb = a.q_abs ? (int64_t)((d.rp + 63) / 64) * d.heads * ((a.tokens + 15) / 16) : 0;
        const dim3 grid((unsigned)(a.tokens + absorb));
        if (dtype) latent_append_few_kernel<float><<<grid, 256, 0, stream>>>(a, d);
        else latent_append_few_kernel<uint16_t><<<grid, 256, 0, stream>>>(a, d);
    } else {
        const dim3 grid((unsigned)((a.tokens + 3) / 4));
        if (dtype) latent_append_kernel<float><<<grid, 256, 0, stream>>>(a, d);
        else latent_append_kernel<uint16_t><<<grid, 256, 0, stream>>>(a, d);
    }
}

// 1024 latent columns: two 32-row tiles of them are 130 KiB of LDS, the scores 9 KiB
bool latent_rows_mfma_supported(const LatentDims& d) { return d.rp <= 1024 && d.dr <= 64; }

int64_t latent_rows_workspace_floats(const LatentDims& d, int64_t tokens, int nsplit) {
    return tokens * d.heads * nsplit * (d.rp + 4);
}

void launch_latent_rows_mfma(const LatentRowsArgs& a, const LatentDims& d, hipStream_t stream) {
    const int64_t tokens = (int64_t)a.batch * a.seq;
    if (d.rp <= 64) partial_t<1>(a, d, stream);
    else if (d.rp <= 128) partial_t<2>(a, d, stream);
    else if (d.rp <= 256) partial_t<4>(a, d, stream);
    else if (d.rp <= 384) partial_t<6>(a, d, stream);
    else if (d.rp <= 512) partial_t<8>(a, d, stream);
    else partial_t<16>(a, d, stream);
    latent_merge_kernel<<<(unsigned)(tokens * d.heads), 128, 0, stream>>>(a, d);
    latent_expand_kernel<<<dim3((unsigned)(d.vp / 16), (unsigned)d.heads, (unsigned)((tokens + 15) / 16)), 256, 0,
                           stream>>>(a, d);
}

bool latent_rows_general_supported(const LatentDims& d) { return d.rp <= kGenRank && d.dr <= kGenDims; }

void launch_latent_rows_general(const LatentRowsArgs& a, const LatentDims& d, int dtype, hipStream_t stream) {
    const dim3 grid((unsigned)((int64_t)a.batch * a.seq), (unsigned)d.heads);
    if (dtype) latent_general_kernel<float><<<grid, 256, 0, stream>>>(a, d);
    else latent_general_kernel<uint16_t><<<grid, 256, 0, stream>>>(a, d);
}

}  // namespace astrai_mix
