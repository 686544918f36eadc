// Latent attention, everything but the prompt kernel: per-head keys and values are projections
// W_uk c, W_uv c of a cached latent c, plus one rotated key part shared by all heads.
//
//   latent_append   rotates the queries' rotated parts in place, norms the new latents, rotates
//                   the new key parts and writes both into the cache
//   rows path       a few new tokens against the cache without ever forming keys or values:
//                   q_u . (W_uk c) = (W_uk^T q_u) . c, and the output is W_uv (sum p c). With the
//                   projection absorbed into the query, all heads of a token share one key/value
//                   row per position, so the cache is read once per 16 (token, head) rows.
//     absorb          q_abs[t, h] = W_uk[h]^T q_u[t, h]            (MFMA, weight-streaming)
//     partial         split-context attention in the latent space  (MFMA)
//     merge + expand  splits merged, W_uv[h] applied, output gate   (MFMA, weight-streaming)
//   general path    the same three steps on the vector ALU for any size and for float
#include "mix_common.cuh"
#include "mix_launchers.h"

namespace astrai_mix {

namespace {

// ---- append: one wave per token -----------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void latent_append_kernel(LatentAppendArgs a, LatentDims d) {
    const int lane = threadIdx.x & 63;
    const int64_t t = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t >= a.tokens) return;
    const int64_t b = t / a.seq;
    const int64_t pos = a.positions[t - b * a.seq];
    if (pos < 0 || pos >= a.max_len || pos >= a.rot_rows) return;
    T* row = static_cast<T*>(a.proj) + t * a.ld;
    const float2* rot = reinterpret_cast<const float2*>(a.rot) + pos * a.half;
    const int qs = d.dn + d.dr;
    for (int i = lane; i < d.heads * a.half; i += 64) {
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
    for (int c = lane * 4; c < d.rp; c += 256) {
        const f32x4 v = Elem<T>::get4(src + c);
        s += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
    }
    const float r = 1.0f / sqrtf(wave_sum(s) / (float)a.kv_rank + a.eps);
    for (int c = lane * 4; c < d.rp; c += 256) {
        f32x4 v = Elem<T>::get4(src + c);
        const f32x4 w = *reinterpret_cast<const f32x4*>(a.norm_w + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = v[e] * r * w[e];
        Elem<T>::put4(dst + c, v);
    }
    src += d.rp;
    dst += d.rp;
    for (int p = lane; p < a.half; p += 64) {
        const float2 cs = rot[p];
        const float x = Elem<T>::get(src + p), y = Elem<T>::get(src + p + a.half);
        Elem<T>::put(dst + p, x * cs.x - y * cs.y);
        Elem<T>::put(dst + p + a.half, y * cs.x + x * cs.y);
    }
    for (int p = 2 * a.half + lane; p < d.dr; p += 64) dst[p] = src[p];
}

// ---- absorb (bf16): q_abs[t, h, r] = sum_d q[t, h, d] w_uk_t[h, r, d] ------------------------------
// One workgroup per (64 latent columns, head, 16 tokens), a wave per 16 columns. Weight rows are the
// MFMA's rows and tokens its columns, so a lane ends up with four consecutive latent columns of one
// token. Both operands come straight from memory, 16 bytes a lane.
__global__ __launch_bounds__(256) void latent_absorb_kernel(LatentRowsArgs a, LatentDims d) {
    const int lane = threadIdx.x & 63, c16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int r0 = (int)blockIdx.x * 64 + wave * 16;
    if (r0 >= d.rp) return;
    const int h = blockIdx.y;
    const int64_t tokens = (int64_t)a.batch * a.seq;
    const int64_t t = (int64_t)blockIdx.z * 16 + c16;
    const bool live = t < tokens;
    const uint16_t* q = static_cast<const uint16_t*>(a.proj) + (live ? t : 0) * a.ld + h * (d.dn + d.dr) + 8 * g;
    const uint16_t* w = static_cast<const uint16_t*>(a.w_uk_t) + ((int64_t)h * d.rp + r0 + c16) * d.dn + 8 * g;
    f32x4 acc = {0, 0, 0, 0};
    for (int k = 0; k < d.dn; k += 32) {
        const u32x4 wf = *reinterpret_cast<const u32x4*>(w + k);
        const u32x4 qf = live ? *reinterpret_cast<const u32x4*>(q + k) : u32x4{0, 0, 0, 0};
        acc = mfma16(wf, qf, acc);
    }
    if (live)
        Elem<uint16_t>::put4(static_cast<uint16_t*>(a.q_abs) + (t * d.heads + h) * d.rp + r0 + 4 * g, acc);
}

// ---- split-context attention over the latent rows (bf16) -------------------------------------------
// Rows are (token, head) pairs of one sequence, token-major; a workgroup takes 16 of them and one
// split of the keys, in tiles of 32. Four waves:
//   scores   wave (kh, ch) multiplies keys 16 kh .. of the tile with half ch of the row's 32-element
//            steps; its key operand comes straight from the cache, and the same registers are
//            written to LDS for the value product. The two halves meet in LDS.
//   softmax  fp32, every wave for itself: lane (query c16, group g) holds keys 8g .. 8g+7, which is
//            the value product's operand layout. Probabilities go in as two bf16 terms.
//   values   wave w accumulates latent columns 16 (w + 4 i) .., the transposed operand out of LDS.
// The LDS tiles alternate between two buffers: one barrier per tile.
// KS: steps per half (compile time), also the bound on a wave's column tiles.
template <int KS>
__global__ __launch_bounds__(256) void latent_partial_kernel(LatentRowsArgs a, LatentDims d) {
    constexpr int kScRow = 36;                       // floats per query row of scores (32 + padding)
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    const int lane = threadIdx.x & 63, c16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int kh = wave & 1, ch = wave >> 1;
    const int split = blockIdx.x, rt = blockIdx.y, b = blockIdx.z;
    const int rows = a.seq * d.heads;
    const int vrow = d.rp * 2 + 32;                  // bytes per latent row in LDS
    uint8_t* vt = lds;
    float* sc = reinterpret_cast<float*>(lds + 2 * 32 * vrow);

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

    const int64_t ldc = d.rp + d.dr;
    const int steps = (int)(ldc >> 5);
    const int half_steps = (steps + 1) >> 1;
    const int st0 = ch * half_steps, nst = min(half_steps, steps - st0);
    // query operand of this wave's steps
    u32x4 qf[KS];
    {
        const int64_t t = (int64_t)b * a.seq + tok;
        const uint16_t* qa = static_cast<const uint16_t*>(a.q_abs) + (t * d.heads + head) * d.rp;
        const uint16_t* qr = static_cast<const uint16_t*>(a.proj) + t * a.ld + head * (d.dn + d.dr) + d.dn - d.rp;
#pragma unroll
        for (int i = 0; i < KS; ++i) {
            const int e = (st0 + i) * 32 + 8 * g;
            qf[i] = (i < nst && live) ? *reinterpret_cast<const u32x4*>((e < d.rp ? qa : qr) + e) : u32x4{0, 0, 0, 0};
        }
    }
    const uint16_t* cache = static_cast<const uint16_t*>(a.cache) + (int64_t)b * a.max_len * ldc + st0 * 32 + 8 * g;
    u32x4 kf[KS];
    auto fetch = [&](int t) {
        const int key = kmin + t * 32 + kh * 16 + c16;
        const bool ok = t < t1 && key <= kmax;
        const uint16_t* p = cache + (int64_t)(ok ? key : 0) * ldc;
#pragma unroll
        for (int i = 0; i < KS; ++i)
            kf[i] = (ok && i < nst) ? *reinterpret_cast<const u32x4*>(p + i * 32) : u32x4{0, 0, 0, 0};
    };
    fetch(t0);

    f32x4 acc[KS];
#pragma unroll
    for (int i = 0; i < KS; ++i) acc[i] = f32x4{0, 0, 0, 0};
    float m = kNegBig, l = 0.0f;
    const float c = d.scale * kLog2e;
    const int rtiles = d.rp >> 4;
    int buf = 0;
    for (int t = t0; t < t1; ++t, buf ^= 1) {
        uint8_t* v = vt + buf * 32 * vrow;
        float* s = sc + buf * 2 * 16 * kScRow;
        f32x4 part = {0, 0, 0, 0};
#pragma unroll
        for (int i = 0; i < KS; ++i) {
            if (i < nst) {
                part = mfma16(kf[i], qf[i], part);
                const int e = (st0 + i) * 32 + 8 * g;
                if (e < d.rp) *reinterpret_cast<u32x4*>(v + (kh * 16 + c16) * vrow + e * 2) = kf[i];
            }
        }
        *reinterpret_cast<f32x4*>(s + (ch * 16 + c16) * kScRow + kh * 16 + 4 * g) = part;
        fetch(t + 1);
        __syncthreads();
        float p[8], tm = kNegBig;
        {
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
        }
        tm = fmaxf(tm, __shfl_xor(tm, 16, kWave));
        tm = fmaxf(tm, __shfl_xor(tm, 32, kWave));
        const float m_new = fmaxf(m, tm);
        const float alpha = __builtin_amdgcn_exp2f(m - m_new);
        m = m_new;
        float ps = 0.0f;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            p[e] = p[e] > 0.5f * kNegBig ? __builtin_amdgcn_exp2f(p[e] - m_new) : 0.0f;
            ps += p[e];
        }
        ps += __shfl_xor(ps, 16, kWave);
        ps += __shfl_xor(ps, 32, kWave);
        l = l * alpha + ps;
        u32x4 hi, lo;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            uint32_t h2, l2;
            split2(p[2 * e], p[2 * e + 1], h2, l2);
            hi[e] = h2;
            lo[e] = l2;
        }
        // transposed latent operand: 16 columns x 32 keys, lane group g takes keys 8g .. 8g+7
        const uint8_t* src = v + (8 * g + (c16 >> 2)) * vrow + (c16 & 3) * 8;
#pragma unroll
        for (int i = 0; i < KS; ++i) {
            const int rti = wave + 4 * i;
            if (rti < rtiles) {
                const uint8_t* q = src + rti * 32;
                const u32x4 vf = join(lds_read_tr(q), lds_read_tr(q + 4 * vrow));
                f32x4 o = acc[i];
#pragma unroll
                for (int e = 0; e < 4; ++e) o[e] *= alpha;
                o = mfma16(vf, hi, o);
                acc[i] = mfma16(vf, lo, o);
            }
        }
    }
    if (!live) return;
    // workspace per (row, split): rp values, then maximum and sum
    float* w = a.ws + (((int64_t)b * rows + row) * a.nsplit + split) * (d.rp + 4);
#pragma unroll
    for (int i = 0; i < KS; ++i) {
        const int rti = wave + 4 * i;
        if (rti < rtiles) *reinterpret_cast<f32x4*>(w + rti * 16 + 4 * g) = acc[i];
    }
    if (wave == 0 && g == 0) {
        w[d.rp] = m;
        w[d.rp + 1] = l;
    }
}

// ---- merge the splits, apply W_uv, gate (bf16) -------------------------------------------------------
// One workgroup per (64 value columns, head, 16 tokens). Sixteen threads merge a token's splits
// into LDS as bf16; then a wave per 16 value columns, as in absorb.
constexpr int kMaxSplit = 64;

__global__ __launch_bounds__(256) void latent_expand_kernel(LatentRowsArgs a, LatentDims d) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    __shared__ float wt[16][kMaxSplit];
    const int tid = threadIdx.x;
    const int h = blockIdx.y;
    const int64_t tokens = (int64_t)a.batch * a.seq;
    const int orow = d.rp * 2 + 16;
    {
        const int i = tid >> 4, j = tid & 15;
        const int64_t t = (int64_t)blockIdx.z * 16 + i;
        const bool live = t < tokens;
        const int64_t base = ((live ? t : 0) * d.heads + h) * a.nsplit;
        const float* w = a.ws + base * (d.rp + 4);
        float big = kNegBig, sum = 0.0f;
        for (int s = 0; s < a.nsplit; ++s) big = fmaxf(big, w[(int64_t)s * (d.rp + 4) + d.rp]);
        for (int s = 0; s < a.nsplit; ++s) {
            const float* e = w + (int64_t)s * (d.rp + 4) + d.rp;
            sum += e[1] * __builtin_amdgcn_exp2f(e[0] - big);
        }
        const float inv = (live && sum > 0.0f) ? 1.0f / sum : 0.0f;
        for (int s = j; s < a.nsplit; s += 16)
            wt[i][s] = __builtin_amdgcn_exp2f(w[(int64_t)s * (d.rp + 4) + d.rp] - big) * inv;
        __syncthreads();
        for (int r = j * 4; r < d.rp; r += 64) {
            f32x4 o = {0, 0, 0, 0};
            for (int s = 0; s < a.nsplit; ++s) {
                const f32x4 v = *reinterpret_cast<const f32x4*>(w + (int64_t)s * (d.rp + 4) + r);
                const float f = wt[i][s];
#pragma unroll
                for (int e = 0; e < 4; ++e) o[e] += f * v[e];
            }
            Elem<uint16_t>::put4(reinterpret_cast<uint16_t*>(lds + i * orow) + r, o);
        }
        __syncthreads();
    }
    const int lane = tid & 63, c16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int v0 = (int)blockIdx.x * 64 + wave * 16;
    if (v0 >= d.vp) return;
    const uint16_t* w = static_cast<const uint16_t*>(a.w_ukv) +
                        ((int64_t)h * (d.dn + d.vp) + d.dn + v0 + c16) * d.rp + 8 * g;
    const uint8_t* o = lds + c16 * orow + 16 * g;
    f32x4 acc = {0, 0, 0, 0};
    for (int k = 0; k < d.rp; k += 32)
        acc = mfma16(*reinterpret_cast<const u32x4*>(w + k), *reinterpret_cast<const u32x4*>(o + k * 2), acc);
    const int64_t t = (int64_t)blockIdx.z * 16 + c16;
    if (t >= tokens) return;
    const float gate = sigmoid(Elem<uint16_t>::get(static_cast<const uint16_t*>(a.proj) + t * a.ld + a.g_off + h));
#pragma unroll
    for (int e = 0; e < 4; ++e) acc[e] *= gate;
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

template <int KS>
void partial_t(const LatentRowsArgs& a, const LatentDims& d, hipStream_t stream) {
    const int rows = a.seq * d.heads;
    const size_t shared = 2 * 32 * (size_t)(d.rp * 2 + 32) + 2 * 2 * 16 * 36 * sizeof(float);
    static const hipError_t once = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_partial_kernel<KS>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    (void)once;
    const dim3 grid((unsigned)a.nsplit, (unsigned)((rows + 15) / 16), (unsigned)a.batch);
    latent_partial_kernel<KS><<<grid, 256, shared, stream>>>(a, d);
}

}  // namespace

void launch_latent_append(const LatentAppendArgs& a, const LatentDims& d, int dtype, hipStream_t stream) {
    const dim3 grid((unsigned)((a.tokens + 3) / 4));
    if (dtype) latent_append_kernel<float><<<grid, 256, 0, stream>>>(a, d);
    else latent_append_kernel<uint16_t><<<grid, 256, 0, stream>>>(a, d);
}

// 1024 latent columns: two 32-row tiles of them are 130 KiB of LDS, the scores 9 KiB
bool latent_rows_mfma_supported(const LatentDims& d) { return d.rp <= 1024 && d.rp + d.dr <= 1152; }

int64_t latent_rows_workspace_floats(const LatentDims& d, int64_t tokens, int nsplit) {
    return tokens * d.heads * nsplit * (d.rp + 4);
}

void launch_latent_rows_mfma(const LatentRowsArgs& a, const LatentDims& d, hipStream_t stream) {
    const unsigned tt = (unsigned)(((int64_t)a.batch * a.seq + 15) / 16);
    latent_absorb_kernel<<<dim3((unsigned)((d.rp + 63) / 64), (unsigned)d.heads, tt), 256, 0, stream>>>(a, d);
    const int half = ((d.rp + d.dr) / 32 + 1) / 2;
    if (half <= 2) partial_t<2>(a, d, stream);
    else if (half <= 4) partial_t<4>(a, d, stream);
    else if (half <= 6) partial_t<6>(a, d, stream);
    else if (half <= 10) partial_t<10>(a, d, stream);
    else partial_t<18>(a, d, stream);
    const size_t shared = 16 * (size_t)(d.rp * 2 + 16);
    latent_expand_kernel<<<dim3((unsigned)((d.vp + 63) / 64), (unsigned)d.heads, tt), 256, shared, stream>>>(a, d);
}

bool latent_rows_general_supported(const LatentDims& d) { return d.rp <= kGenRank && d.dr <= kGenDims; }

void launch_latent_rows_general(const LatentRowsArgs& a, const LatentDims& d, int dtype, hipStream_t stream) {
    const dim3 grid((unsigned)((int64_t)a.batch * a.seq), (unsigned)d.heads);
    if (dtype) latent_general_kernel<float><<<grid, 256, 0, stream>>>(a, d);
    else latent_general_kernel<uint16_t><<<grid, 256, 0, stream>>>(a, d);
}

}  // namespace astrai_mix
