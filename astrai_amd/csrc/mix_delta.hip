// Gated delta rule with one decay per key channel: per head, with unit k, scaled unit q,
//   S <- diag(g_t) S,   u_t = beta_t (v_t - S^T k_t),   S <- S + k_t u_t^T,   o_t = S^T q_t,
// g = exp(-exp(A) softplus(z + dt_bias)) per key channel, beta a sigmoid, S fp32 [dp, vp].
//
// Chunked form (prompts, bf16), chunks of 16 tokens. With G_t the product of the decays of the chunk up to
// token t and L_tj = product of the decays of tokens j + 1 .. t (all per channel, all <= 1):
//   M_tj = beta_t sum_d k_td L_tjd k_jd (j < t),        P_tj = sum_d q_td L_tjd k_jd (j <= t),
//   U = (I + M)^-1 diag(beta) (V - (G K) S),            O = (G Q) S + P U,
//   S_new = diag(G_15) S + (L_15 K)^T U.
//   prep   every chunk of every head at once: everything but S and V, written as MFMA operand fragments
//          (the "image"). L cannot be split into a factor of t and one of j against the chunk's start (the
//          second would overflow under strong decays), so pairs are grouped by the highest bit in which t
//          and j differ: with m the middle of their common block of 2, 4, 8 or 16 tokens, L_tj is
//          (decays m .. t)(decays j + 1 .. m - 1), both <= 1. One wave per such level and product.
//   walk   chunk after chunk per head; a wave owns 16 or 32 value columns and all key channels, S in fp32
//          accumulators. With value columns as MFMA columns throughout, every accumulator (S, V - Y, U) is
//          the next product's operand already; images stream into LDS by direct loads, one chunk ahead.
// 32-bit factors enter the matrix cores as two bf16 terms; a 16-deep contraction uses the two halves of a
// 32-deep MFMA for the two terms of its left factor.
//
// Step kernel (decoding, and everything in float): token by token, the state in registers, one workgroup per
// head; norm and output gate in its epilogue. For a few tokens it also convolves its inputs.
#include <type_traits>

#include "mix_conv.cuh"
#include "mix_launchers.h"

namespace astrai_mix {

namespace {

constexpr int kC = kDeltaChunk;
constexpr float kUnitEps = 1e-6f;

// ---- step ---------------------------------------------------------------------------------------
constexpr int kStepThreads = 512, kStepWaves = kStepThreads / 64;

// thread (rg, vq): value columns 4 vq .., state rows rg + RG i; vq runs over vqp = a power of two >= vp / 4
template <typename T, int NR, bool FUSED>
__global__ __launch_bounds__(kStepThreads, NR <= 8 ? 4 : 2) void delta_step_kernel(DeltaArgs a, int vqp) {
    extern __shared__ __attribute__((aligned(16))) float sh[];
    const int rgs = kStepThreads / vqp, rows = rgs * NR;   // rows >= dp, those past it zero
    float* const qs = sh;                   // [rows]
    float* const ks = qs + rows;            // [rows]
    float* const gs = ks + rows;            // [rows]
    float* const vs = gs + rows;            // [vp]
    float* const red = vs + a.vp;           // [2][kStepWaves][vqp * 4]
    float* const redk = red + 2 * kStepWaves * vqp * 4;   // [kStepWaves]
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int h = blockIdx.x, b = blockIdx.y, grp = h / (a.heads / a.kv_heads);
    const int rg = tid / vqp, vq = tid % vqp;
    const bool v_live = vq * 4 < a.vp;
    const int q_col = grp * a.dp, k_col = a.kv_heads * a.dp + grp * a.dp, v_col = 2 * a.kv_heads * a.dp + h * a.vp;
    const int64_t start = FUSED ? a.conv.positions[0] : 0;
    float* state = a.state + ((int64_t)b * a.heads + h) * a.dp * a.vp;
    f32x4 s[NR];
#pragma unroll
    for (int i = 0; i < NR; ++i) {
        const int r = rg + rgs * i;
        s[i] = (v_live && r < a.dp) ? *reinterpret_cast<const f32x4*>(state + (int64_t)r * a.vp + vq * 4) : f32x4{0, 0, 0, 0};
    }
    for (int r = a.dp + tid; r < rows; r += kStepThreads) qs[r] = ks[r] = gs[r] = 0.0f;
    const float decay = a.decay[h];
    for (int t = 0; t < a.seq; ++t) {
        const int64_t row = (int64_t)b * a.seq + t;
        auto input4 = [&](int c) -> f32x4 {
            if constexpr (FUSED) {
                f32x4 x = conv_at4<T>(a.conv, b, start, t, c);
#pragma unroll
                for (int e = 0; e < 4; ++e) x[e] = rounded<T>(silu_as<T>(x[e]));
                return x;
            } else {
                return Elem<T>::get4(static_cast<const T*>(a.qkv) + row * a.ldq + c);
            }
        };
        // wave 0: q, wave 1: k (unit vectors), waves 2, 3: decays, the others: v
        if (wave < 2) {
            float* dst = wave ? ks : qs;
            float sq = 0.0f;
            for (int c = lane * 4; c < a.dp; c += 256) {
                const f32x4 x = input4((wave ? k_col : q_col) + c);
                sq += (x[0] * x[0] + x[1] * x[1]) + (x[2] * x[2] + x[3] * x[3]);
                *reinterpret_cast<f32x4*>(dst + c) = x;
            }
            const float f = (wave ? 1.0f : a.q_scale) / sqrtf(wave_sum(sq) + kUnitEps);
            for (int c = lane * 4; c < a.dp; c += 256) {   // (each lane what it wrote)
                f32x4 x = *reinterpret_cast<const f32x4*>(dst + c);
#pragma unroll
                for (int e = 0; e < 4; ++e) x[e] *= f;
                *reinterpret_cast<f32x4*>(dst + c) = x;
            }
        } else if (wave < 4) {
            for (int c = (wave - 2) * 64 + lane; c < a.dp; c += 128) {
                const float z = a.z[row * a.heads * a.dp + h * a.dp + c] + a.dt_bias[h * a.dp + c];
                const float x = -decay * softplus_as<T>(z);
                gs[c] = sizeof(T) == 2 ? __builtin_amdgcn_exp2f(kLog2e * x) : expf(x);
            }
        } else {
            for (int c = ((wave - 4) * 64 + lane) * 4; c < a.vp; c += 1024) *reinterpret_cast<f32x4*>(vs + c) = input4(v_col + c);
        }
        __syncthreads();
        f32x4 pk = {0, 0, 0, 0}, pq = {0, 0, 0, 0};
        float kq = 0.0f;
#pragma unroll
        for (int i = 0; i < NR; ++i) {
            const int r = rg + rgs * i;
            const float g = gs[r], k = ks[r], q = qs[r];
            kq = fmaf(k, q, kq);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                s[i][e] *= g;
                pk[e] = fmaf(s[i][e], k, pk[e]);
                pq[e] = fmaf(s[i][e], q, pq[e]);
            }
        }
        for (int off = vqp; off < kWave; off <<= 1) {
            kq += __shfl_xor(kq, off, kWave);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                pk[e] += __shfl_xor(pk[e], off, kWave);
                pq[e] += __shfl_xor(pq[e], off, kWave);
            }
        }
        // (a wave with vqp = 64 holds one row group)
        if (lane < vqp) {
            *reinterpret_cast<f32x4*>(red + (wave * vqp + vq) * 4) = pk;
            *reinterpret_cast<f32x4*>(red + ((kStepWaves + wave) * vqp + vq) * 4) = pq;
        }
        if (lane == 0) redk[wave] = kq;
        __syncthreads();
        f32x4 o = {0, 0, 0, 0}, u = {0, 0, 0, 0};
        kq = 0.0f;
#pragma unroll 2
        for (int w = 0; w < kStepWaves; ++w) {
            u += *reinterpret_cast<const f32x4*>(red + (w * vqp + vq) * 4);
            o += *reinterpret_cast<const f32x4*>(red + ((kStepWaves + w) * vqp + vq) * 4);
            kq += redk[w];
        }
        const float beta = sigmoid(Elem<T>::get(static_cast<const T*>(a.proj) + row * a.ld + a.b_off + h));
        const f32x4 v = v_live ? *reinterpret_cast<const f32x4*>(vs + vq * 4) : f32x4{0, 0, 0, 0};
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            u[e] = beta * (v[e] - u[e]);
            o[e] = fmaf(u[e], kq, o[e]);
        }
#pragma unroll
        for (int i = 0; i < NR; ++i) {
            const float k = ks[rg + rgs * i];
#pragma unroll
            for (int e = 0; e < 4; ++e) s[i][e] = fmaf(k, u[e], s[i][e]);
        }
        if (rg == 0) {   // the first vqp lanes of wave 0
            float sq = v_live ? (o[0] * o[0] + o[1] * o[1]) + (o[2] * o[2] + o[3] * o[3]) : 0.0f;
            for (int off = vqp / 2; off; off >>= 1) sq += __shfl_xor(sq, off, kWave);
            if (v_live) {
                const float f = 1.0f / sqrtf(sq / (float)a.vdim + a.eps);
                const int c = h * a.vp + vq * 4;
                const f32x4 z = Elem<T>::get4(static_cast<const T*>(a.gate) + row * a.ldg + c);
                const f32x4 w = *reinterpret_cast<const f32x4*>(a.norm_w + vq * 4);
#pragma unroll
                for (int e = 0; e < 4; ++e) o[e] = o[e] * f * w[e] * sigmoid(z[e]);
                Elem<T>::put4(static_cast<T*>(a.out) + row * a.heads * a.vp + c, o);
            }
        }
        __syncthreads();   // vectors and partial sums of this token are no longer read
    }
#pragma unroll
    for (int i = 0; i < NR; ++i) {
        const int r = rg + rgs * i;
        if (v_live && r < a.dp) *reinterpret_cast<f32x4*>(state + (int64_t)r * a.vp + vq * 4) = s[i];
    }
    if constexpr (FUSED) {
        // the last inputs into the ring, rows that no workgroup of this launch reads; a group's first head
        // writes the shared q and k
        const bool first = h % (a.heads / a.kv_heads) == 0;
        const int n = (first ? 2 * a.dp : 0) + a.vp;
        for (int c = tid * 4; c < n; c += kStepThreads * 4) {
            const int d = first ? c : c + 2 * a.dp;
            const int col = d < a.dp ? q_col + d : d < 2 * a.dp ? k_col + d - a.dp : v_col + d - 2 * a.dp;
            for (int t = max(a.seq - a.conv.taps + 1, 0); t < a.seq; ++t) ring_put4<T>(a.conv, b, start, t, col);
        }
    }
}

// ---- chunk: image of a (sequence, head, chunk), in fragments of 64 lanes x 16 bytes ---------------------
//   [0, NS)       G K, high terms: lane (g, c16), step s: row c16, channels 32 s + 4 g .. and 32 s + 16 + 4 g ..
//   [NS, 2 NS)    its low terms
//   [2 NS, 4 NS)  G Q likewise
//   [4 NS, 6 NS)  (L_15 K)^T: tile i: row = channel 16 i + c16, tokens 4 g .., high terms then low
//   6 NS          (I + M)^-1 diag(beta): row c16, tokens 4 g .., high terms then low
//   6 NS + 1      P likewise
//   then dp floats: G_15
template <int DP>
struct Image {
    static constexpr int NS = DP / 32;
    static constexpr int kFrags = 6 * NS + 2;
    static constexpr int kBytes = kFrags * 1024 + DP * 4;
    static constexpr int kDma = (kBytes + 1023) / 1024;    // 1 KiB pieces; memory per image is whole pieces
};

__device__ __forceinline__ u32x4 split4(f32x4 v) {   // four high terms, four low terms
    uint32_t h0, l0, h1, l1;
    split2(v[0], v[1], h0, l0);
    split2(v[2], v[3], h1, l1);
    return u32x4{h0, h1, l0, l1};
}

constexpr int kPrepThreads = 512;

// Thread roles: a pair of channels, keys or queries, eight of the 16 tokens, one of two levels at a time. A level's
// matrices hold the factors of keys for all tokens and of queries for the upper ones; the levels are done in two rounds
// of two, so that four workgroups fit a CU.
template <int DP>
__global__ __launch_bounds__(kPrepThreads, DP <= 128 ? 8 : 2) void delta_prep_kernel(DeltaArgs a, int chunks) {
    constexpr int NS = DP / 32, kRow = DP * 2 + 16, kMat = kC * kRow;   // bytes
    constexpr int kPairs = DP / 2, kPer = (kPairs + 63) / 64;           // channel pairs, of a thread
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    constexpr int kHalfMat = kMat / 2, kLevel = 2 * kMat + 2 * kHalfMat;
    uint8_t* const mats = lds;                    // [2 levels][k hi, k lo: kC rows; q hi, q lo: kC / 2 rows][kRow]
    float* const lg = reinterpret_cast<float*>(lds + 2 * kLevel);   // [kC][DP] decays
    float* const inv = lg + kC * DP;              // [2][kC]: factor of k, of q
    float* const diag = inv + 2 * kC;             // [kC]
    float* const beta = diag + kC;                // [kC]
    float* const ms = beta + kC;                  // [kC][20]
    float* const ps = ms + kC * 20;               // [kC][20]
    const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int chunk = blockIdx.x, h = blockIdx.y, b = blockIdx.z, grp = h / (a.heads / a.kv_heads);
    const int t0 = chunk * kC, n = min(kC, a.seq - t0);
    const int64_t row0 = (int64_t)b * a.seq + t0;
    const uint16_t* q = static_cast<const uint16_t*>(a.qkv) + row0 * a.ldq + grp * a.dp;
    const uint16_t* k = q + a.kv_heads * a.dp;
    uint8_t* image = static_cast<uint8_t*>(a.image) + (((int64_t)b * a.heads + h) * chunks + chunk) * (Image<DP>::kDma * 1024);

    // the first half: norms, 16 lanes per token, which also give q . k of the same token
    if (wave < 4) {
        const int t = tid >> 4, l = tid & 15;
        float sq = 0.0f, sk = 0.0f, qk = 0.0f;
        if (t < n)
            for (int c = l * 8; c < a.dp; c += 128) {
                float x[8], y[8];
                w8a8::unpack8(*reinterpret_cast<const u32x4*>(q + (int64_t)t * a.ldq + c), x);
                w8a8::unpack8(*reinterpret_cast<const u32x4*>(k + (int64_t)t * a.ldq + c), y);
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    sq = fmaf(x[e], x[e], sq);
                    sk = fmaf(y[e], y[e], sk);
                    qk = fmaf(x[e], y[e], qk);
                }
            }
#pragma unroll
        for (int off = 8; off; off >>= 1) {
            sq += __shfl_xor(sq, off, kWave);
            sk += __shfl_xor(sk, off, kWave);
            qk += __shfl_xor(qk, off, kWave);
        }
        if (l == 0) {
            const float fq = a.q_scale / sqrtf(sq + kUnitEps), fk = 1.0f / sqrtf(sk + kUnitEps);
            inv[t] = fk;
            inv[kC + t] = fq;
            diag[t] = qk * fq * fk;
            beta[t] = t < n ? sigmoid(Elem<uint16_t>::get(static_cast<const uint16_t*>(a.proj) + (row0 + t) * a.ld + a.b_off + h))
                            : 0.0f;
        }
    }
    // decays, four channels at a time
    {
        const float decay = -kLog2e * a.decay[h];
        const float* z = a.z + row0 * a.heads * a.dp + h * a.dp;
        for (int i = tid; i < kC * (DP / 4); i += kPrepThreads) {
            const int t = i / (DP / 4), d = i % (DP / 4) * 4;
            f32x4 x = {1, 1, 1, 1};
            if (t < n && d < a.dp) {
                const f32x4 zz = *reinterpret_cast<const f32x4*>(z + (int64_t)t * a.heads * a.dp + d);
                const f32x4 bias = *reinterpret_cast<const f32x4*>(a.dt_bias + h * a.dp + d);
#pragma unroll
                for (int e = 0; e < 4; ++e) x[e] = __builtin_amdgcn_exp2f(decay * softplus_fast(zz[e] + bias[e]));
            }
            *reinterpret_cast<f32x4*>(lg + t * DP + d) = x;
        }
    }
    const bool is_q = wave >= 4;
    const int half = wave & 1, sel = (wave >> 1) & 1, r0 = half * 8;   // tokens r0 .. r0 + 7
    f32x2 x[kPer][8];    // this pair's unit vectors
    const uint16_t* src = is_q ? q : k;
#pragma unroll
    for (int p = 0; p < kPer; ++p) {
        const int d = (lane + p * 64) * 2;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const int t = r0 + i;
            const uint32_t raw = (t < n && d < a.dp) ? *reinterpret_cast<const uint32_t*>(src + (int64_t)t * a.ldq + d) : 0;
            x[p][i] = f32x2{__uint_as_float(raw << 16), __uint_as_float(raw & 0xffff0000u)};
        }
    }
    __syncthreads();
    auto scale = [](f32x2 u, f32x2 v) { return f32x2{u[0] * v[0], u[1] * v[1]}; };
    // both terms of a pair, the low ones `dist` bytes further
    auto put = [&](uint8_t* hi, int dist, int off, f32x2 v) {
        uint32_t h2, l2;
        split2(v[0], v[1], h2, l2);
        *reinterpret_cast<uint32_t*>(hi + off) = h2;
        *reinterpret_cast<uint32_t*>(hi + dist + off) = l2;
    };
#pragma unroll
    for (int p = 0; p < kPer; ++p)
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const float f = inv[(is_q ? kC : 0) + r0 + i];
            x[p][i] = scale(x[p][i], f32x2{f, f});
        }
#pragma unroll
    for (int round = 0; round < 2; ++round) {
        if (round) __syncthreads();   // the first round's matrices are no longer read
        uint8_t* const lv = mats + sel * kLevel;
#pragma unroll
        for (int p = 0; p < kPer; ++p) {
            const int d = (lane + p * 64) * 2;
            if (d >= DP) continue;
            f32x2 dec[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) dec[i] = *reinterpret_cast<const f32x2*>(lg + (r0 + i) * DP + d);
            // Tokens M .. M + HB - 1 of this half as a block's upper ones: they take the decays M .. t. Their rank
            // among the level's upper tokens is the row of a query.
            auto upper = [&](auto hb, auto m) {
                f32x2 w = {1.0f, 1.0f};
#pragma unroll
                for (int i = m; i < m + hb; ++i) {
                    w = scale(w, dec[i]);
                    const f32x2 v = scale(x[p][i], w);
                    const int t = r0 + i, rank = (t / (2 * hb)) * hb + t % hb;
                    if (is_q) put(lv + 2 * kMat, kHalfMat, rank * kRow + d * 2, v);
                    else put(lv, kMat, t * kRow + d * 2, v);
                }
            };
            // the HB tokens before the middle M as its lower ones (keys): decays j + 1 .. M - 1
            auto lower = [&](auto hb, auto m) {
                if (is_q) return;
                f32x2 w = {1.0f, 1.0f};
#pragma unroll
                for (int i = m - 1; i >= m - hb; --i) {
                    put(lv, kMat, (r0 + i) * kRow + d * 2, scale(x[p][i], w));
                    w = scale(w, dec[i]);
                }
            };
            using std::integral_constant;
            auto block = [&](auto hb, auto m) {
                lower(hb, m);
                upper(hb, m);
            };
            if (round == 0) {
                if (sel == 0) {
                    if (half) upper(integral_constant<int, 8>{}, integral_constant<int, 0>{});
                    else lower(integral_constant<int, 8>{}, integral_constant<int, 8>{});
                } else {
                    block(integral_constant<int, 4>{}, integral_constant<int, 4>{});
                }
            } else if (sel == 0) {
                block(integral_constant<int, 2>{}, integral_constant<int, 2>{});
                block(integral_constant<int, 2>{}, integral_constant<int, 6>{});
            } else {
                block(integral_constant<int, 1>{}, integral_constant<int, 1>{});
                block(integral_constant<int, 1>{}, integral_constant<int, 3>{});
                block(integral_constant<int, 1>{}, integral_constant<int, 5>{});
                block(integral_constant<int, 1>{}, integral_constant<int, 7>{});
            }
            // the last key parts: L_15 K straight into the image
            if (round == sel && !is_q && sel == 1) {
                f32x2 w = {1.0f, 1.0f};
                if (!half) {
#pragma unroll
                    for (int t = kC - 1; t >= 8; --t) w = scale(w, *reinterpret_cast<const f32x2*>(lg + t * DP + d));
                }
                f32x2 v[8];
#pragma unroll
                for (int i = 7; i >= 0; --i) {
                    v[i] = scale(x[p][i], w);
                    w = scale(w, dec[i]);
                }
                uint8_t* dst = image + (4 * NS + (d >> 4)) * 1024 + (d & 15) * 16 + half * 512;
#pragma unroll
                for (int gg = 0; gg < 2; ++gg)
#pragma unroll
                    for (int e = 0; e < 2; ++e)
                        *reinterpret_cast<u32x4*>(dst + gg * 256 + e * 16) =
                            split4(f32x4{v[4 * gg][e], v[4 * gg + 1][e], v[4 * gg + 2][e], v[4 * gg + 3][e]});
                if (!half) *reinterpret_cast<f32x2*>(image + Image<DP>::kFrags * 1024 + d * 4) = w;   // all 16 decays
            }
        }
        __syncthreads();
        // pairs: a wave per level and product (M on the keys' waves, P on the queries'); the level of (t, j) is the
        // highest bit of t ^ j. A lower token's row of P is some upper one's: not used.
        if (half == 0) {
            const int hb = (round ? 2 : 8) >> sel;
            const uint8_t* base = lv + c16 * kRow + 16 * g;
            const uint8_t* left = is_q ? lv + 2 * kMat + ((c16 / (2 * hb)) * hb + c16 % hb) * kRow + 16 * g : base;
            const int dist = is_q ? kHalfMat : kMat;
            f32x4 acc = {0, 0, 0, 0}, acc2 = {0, 0, 0, 0};
#pragma unroll
            for (int s = 0; s < NS; ++s) {
                const u32x4 kh = *reinterpret_cast<const u32x4*>(base + s * 64);
                const u32x4 kl = *reinterpret_cast<const u32x4*>(base + kMat + s * 64);
                const u32x4 lh = *reinterpret_cast<const u32x4*>(left + s * 64);
                const u32x4 ll = *reinterpret_cast<const u32x4*>(left + dist + s * 64);
                acc = mfma16(lh, kh, acc);
                acc2 = mfma16(lh, kl, acc2);
                acc2 = mfma16(ll, kh, acc2);
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int t = 4 * g + e, j = c16, x2 = t ^ j;
                const float v = acc[e] + acc2[e];
                float* dst = (is_q ? ps : ms) + t * 20 + j;
                if (t > j && x2 >= hb && x2 < 2 * hb) *dst = is_q ? v : beta[t] * v;
                else if (round == 0 && sel == 0 && t <= j) *dst = is_q && t == j ? diag[t] : 0.0f;
            }
        }
    }
    __syncthreads();
    // the level matrices are free: G K and G Q go through their place, so that the image leaves in whole pieces
    if (sel == 1) {
#pragma unroll
        for (int p = 0; p < kPer; ++p) {
            const int d = (lane + p * 64) * 2;
            if (d >= DP) continue;
            f32x2 w = {1.0f, 1.0f};
            if (half) {
#pragma unroll
                for (int t = 0; t < 8; ++t) w = scale(w, *reinterpret_cast<const f32x2*>(lg + t * DP + d));
            }
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                w = scale(w, *reinterpret_cast<const f32x2*>(lg + (r0 + i) * DP + d));
                put(mats + (is_q ? 2 : 0) * kMat, kMat, (r0 + i) * kRow + d * 2, scale(x[p][i], w));
            }
        }
    }
    __syncthreads();
    if (wave == 0) {
        // row c16 of X = (I + M)^-1 from X (I + M) = I, last column first
        float y[kC];
#pragma unroll
        for (int j = 0; j < kC; ++j) y[j] = j == c16 ? 1.0f : 0.0f;
#pragma unroll
        for (int s = kC - 1; s >= 1; --s) {
            float m[kC];
#pragma unroll
            for (int j = 0; j < s; j += 4) {
                const f32x4 v = *reinterpret_cast<const f32x4*>(ms + s * 20 + j);
                m[j] = v[0];
                m[j + 1] = v[1];
                m[j + 2] = v[2];
                m[j + 3] = v[3];
            }
#pragma unroll
            for (int j = 0; j < s; ++j) y[j] = fmaf(-y[s], m[j], y[j]);
        }
        f32x4 mine = {0, 0, 0, 0};
#pragma unroll
        for (int gg = 0; gg < 4; ++gg)
            if (g == gg) mine = f32x4{y[4 * gg], y[4 * gg + 1], y[4 * gg + 2], y[4 * gg + 3]};
#pragma unroll
        for (int e = 0; e < 4; ++e) mine[e] *= beta[4 * g + e];
        *reinterpret_cast<u32x4*>(image + 6 * NS * 1024 + lane * 16) = split4(mine);
    } else if (wave == 4) {
        *reinterpret_cast<u32x4*>(image + (6 * NS + 1) * 1024 + lane * 16) =
            split4(*reinterpret_cast<const f32x4*>(ps + c16 * 20 + 4 * g));
    }
    // the other waves: fragments of matrix i / NS, step i % NS
    if (wave == 0 || wave == 4) return;
    for (int i = wave > 4 ? wave - 2 : wave - 1; i < 4 * NS; i += kPrepThreads / 64 - 2) {
        const uint8_t* from = mats + (i / NS) * kMat + c16 * kRow + (i % NS) * 64 + 8 * g;
        *reinterpret_cast<u32x4*>(image + i * 1024 + lane * 16) =
            join(*reinterpret_cast<const u32x2*>(from), *reinterpret_cast<const u32x2*>(from + 32));
    }
}

__device__ __forceinline__ void lds_dma16(__amdgpu_buffer_rsrc_t r, uint8_t* lds_wave_base, uint32_t voff) {
    __builtin_amdgcn_raw_ptr_buffer_load_lds(r, (__attribute__((address_space(3))) void*)lds_wave_base, 16, voff, 0, 0, 0);
}

// VT: 16-column value tiles per wave
template <int DP, int VT>
__global__ __launch_bounds__(256, DP <= 128 ? 2 : 1) void delta_walk_kernel(DeltaArgs a, int chunks) {
    constexpr int NS = DP / 32, NT = DP / 16, kBuf = Image<DP>::kDma * 1024;
    extern __shared__ __attribute__((aligned(1024))) uint8_t lds[];   // two images
    const int tid = threadIdx.x, lane = tid & 63, c16 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int h = blockIdx.y, b = blockIdx.z;
    const int v0 = ((int)blockIdx.x * 4 + wave) * (16 * VT);
    const uint8_t* images = static_cast<const uint8_t*>(a.image) + ((int64_t)b * a.heads + h) * chunks * kBuf;
    auto dma = [&](int c) {
        const __amdgpu_buffer_rsrc_t r = w8a8::make_rsrc(images + (int64_t)c * kBuf, c < chunks ? kBuf : 0);
        uint8_t* dst = lds + (c & 1) * kBuf;
        for (int i = wave; i < Image<DP>::kDma; i += 4) lds_dma16(r, dst + i * 1024, i * 1024 + lane * 16);
    };
    const uint16_t* vsrc = static_cast<const uint16_t*>(a.qkv) + (int64_t)b * a.seq * a.ldq + 2 * a.kv_heads * a.dp + h * a.vp;
    float* state = a.state + ((int64_t)b * a.heads + h) * a.dp * a.vp;
    // S: rows 16 i + 4 g + e, columns v0 + 16 vt + c16
    f32x4 st[NT][VT];
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
        for (int vt = 0; vt < VT; ++vt)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int d = 16 * i + 4 * g + e, v = v0 + 16 * vt + c16;
                st[i][vt][e] = (d < a.dp && v < a.vp) ? state[(int64_t)d * a.vp + v] : 0.0f;
            }
    uint16_t vr[VT][4];
    auto fetch_v = [&](int c) {
#pragma unroll
        for (int vt = 0; vt < VT; ++vt)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int t = c * kC + 4 * g + e, v = v0 + 16 * vt + c16;
                vr[vt][e] = (t < a.seq && v < a.vp) ? vsrc[(int64_t)t * a.ldq + v] : 0;
            }
    };
    f32x4 o[VT];
    auto put_o = [&](int c) {
#pragma unroll
        for (int vt = 0; vt < VT; ++vt)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int t = c * kC + 4 * g + e, v = v0 + 16 * vt + c16;
                if (t < a.seq && v < a.vp)
                    Elem<uint16_t>::put(static_cast<uint16_t*>(a.out) + (((int64_t)b * a.seq + t) * a.heads + h) * a.vp + v, o[vt][e]);
            }
    };
    dma(0);
    fetch_v(0);
    for (int c = 0; c < chunks; ++c) {
        __builtin_amdgcn_s_waitcnt(0x0070);   // vmcnt(0) lgkmcnt(0)
        __syncthreads();                      // image c is there, image c - 1 is no longer read
        if (c) put_o(c - 1);                  // (stores count as outstanding memory operations too: early in the chunk)
        dma(c + 1);
        f32x4 x[VT];
#pragma unroll
        for (int vt = 0; vt < VT; ++vt)
#pragma unroll
            for (int e = 0; e < 4; ++e) x[vt][e] = w8a8::bf16_to_f32(vr[vt][e]);
        fetch_v(c + 1);
        const uint8_t* im = lds + (c & 1) * kBuf;
        auto frag = [&](int i) { return *reinterpret_cast<const u32x4*>(im + i * 1024 + lane * 16); };
        f32x4 y[VT];
#pragma unroll
        for (int vt = 0; vt < VT; ++vt) y[vt] = o[vt] = f32x4{0, 0, 0, 0};
#pragma unroll
        for (int s = 0; s < NS; ++s) {
            const u32x4 kh = frag(s), kl = frag(NS + s), qh = frag(2 * NS + s), ql = frag(3 * NS + s);
#pragma unroll
            for (int vt = 0; vt < VT; ++vt) {
                const u32x4 p0 = split4(st[2 * s][vt]), p1 = split4(st[2 * s + 1][vt]);
                const u32x4 sh = {p0[0], p0[1], p1[0], p1[1]}, sl = {p0[2], p0[3], p1[2], p1[3]};
                y[vt] = mfma16(kh, sh, y[vt]);
                o[vt] = mfma16(qh, sh, o[vt]);
                y[vt] = mfma16(kl, sh, y[vt]);
                o[vt] = mfma16(ql, sh, o[vt]);
                y[vt] = mfma16(kh, sl, y[vt]);
                o[vt] = mfma16(qh, sl, o[vt]);
            }
        }
        const u32x4 tf = frag(6 * NS), pf = frag(6 * NS + 1);
        u32x4 uh[VT], ul[VT];
#pragma unroll
        for (int vt = 0; vt < VT; ++vt) {
            const u32x4 p = split4(x[vt] - y[vt]);
            f32x4 u = {0, 0, 0, 0};
            u = mfma16(tf, u32x4{p[0], p[1], p[0], p[1]}, u);
            u = mfma16(tf, u32x4{p[2], p[3], p[2], p[3]}, u);
            const u32x4 w = split4(u);
            uh[vt] = u32x4{w[0], w[1], w[0], w[1]};
            ul[vt] = u32x4{w[2], w[3], w[2], w[3]};
            o[vt] = mfma16(pf, uh[vt], o[vt]);
            o[vt] = mfma16(pf, ul[vt], o[vt]);
        }
        const float* gam = reinterpret_cast<const float*>(im + Image<DP>::kFrags * 1024) + 4 * g;
#pragma unroll
        for (int i = 0; i < NT; ++i) {
            const f32x4 gg = *reinterpret_cast<const f32x4*>(gam + 16 * i);
            const u32x4 kf = frag(4 * NS + i);
#pragma unroll
            for (int vt = 0; vt < VT; ++vt) {
#pragma unroll
                for (int e = 0; e < 4; ++e) st[i][vt][e] *= gg[e];
                st[i][vt] = mfma16(kf, uh[vt], st[i][vt]);
                st[i][vt] = mfma16(kf, ul[vt], st[i][vt]);
            }
        }
    }
    put_o(chunks - 1);
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
        for (int vt = 0; vt < VT; ++vt)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int d = 16 * i + 4 * g + e, v = v0 + 16 * vt + c16;
                if (d < a.dp && v < a.vp) state[(int64_t)d * a.vp + v] = st[i][vt][e];
            }
}

template <int DP, int VT>
void walk_t(const DeltaArgs& a, int chunks, hipStream_t stream) {
    constexpr int shared = 2 * Image<DP>::kDma * 1024;
    static const hipError_t once = hipFuncSetAttribute(reinterpret_cast<const void*>(&delta_walk_kernel<DP, VT>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, shared);
    (void)once;
    const dim3 grid((unsigned)((a.vp + 64 * VT - 1) / (64 * VT)), (unsigned)a.heads, (unsigned)a.batch);
    delta_walk_kernel<DP, VT><<<grid, 256, shared, stream>>>(a, chunks);
}

template <int DP>
void chunk_t(const DeltaArgs& a, hipStream_t stream) {
    constexpr int shared = 6 * kC * (DP * 2 + 16) + kC * DP * 4 + 4 * kC * 4 + 2 * kC * 20 * 4;
    static const hipError_t once = hipFuncSetAttribute(reinterpret_cast<const void*>(&delta_prep_kernel<DP>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, shared);
    (void)once;
    const int chunks = (a.seq + kC - 1) / kC;
    delta_prep_kernel<DP><<<dim3((unsigned)chunks, (unsigned)a.heads, (unsigned)a.batch), kPrepThreads, shared, stream>>>(a, chunks);
    // wide slices read every image once; narrow ones make more workgroups
    if (DP <= 128 && a.vp > 64 && (int64_t)a.batch * a.heads >= 256) walk_t<DP, 2>(a, chunks, stream);
    else walk_t<DP, 1>(a, chunks, stream);
}

template <typename T, int NR>
void step_n(const DeltaArgs& a, bool fused, int vqp, hipStream_t stream) {
    const int shared = (3 * (kStepThreads / vqp) * NR + a.vp + 2 * kStepWaves * vqp * 4 + kStepWaves) * (int)sizeof(float);
    const dim3 grid((unsigned)a.heads, (unsigned)a.batch);
    if (fused) delta_step_kernel<T, NR, true><<<grid, kStepThreads, shared, stream>>>(a, vqp);
    else delta_step_kernel<T, NR, false><<<grid, kStepThreads, shared, stream>>>(a, vqp);
}

int step_vqp(int vp) {
    int vqp = 8;
    while (vqp * 4 < vp) vqp *= 2;
    return vqp;
}

template <typename T>
void step_t(const DeltaArgs& a, bool fused, hipStream_t stream) {
    const int vqp = step_vqp(a.vp), rows = (a.dp * vqp + kStepThreads - 1) / kStepThreads;
    if (rows <= 4) step_n<T, 4>(a, fused, vqp, stream);
    else if (rows <= 8) step_n<T, 8>(a, fused, vqp, stream);
    else if (rows <= 16) step_n<T, 16>(a, fused, vqp, stream);
    else step_n<T, 32>(a, fused, vqp, stream);
}

}  // namespace

bool delta_step_supported(int dp, int vp) { return vp <= 256 && dp <= 1024 && dp * step_vqp(vp) <= 32 * kStepThreads; }

void launch_delta_step(const DeltaArgs& a, bool fused, int dtype, hipStream_t stream) {
    if (dtype) step_t<float>(a, fused, stream);
    else step_t<uint16_t>(a, fused, stream);
}

bool delta_chunk_supported(int dp, int vp) { return dp <= 256 && vp > 0; }

int64_t delta_image_bytes(int dp) {
    const int kb = dp <= 32 ? Image<32>::kDma : dp <= 64 ? Image<64>::kDma : dp <= 128 ? Image<128>::kDma : Image<256>::kDma;
    return (int64_t)kb * 1024;
}

void launch_delta_chunk(const DeltaArgs& a, hipStream_t stream) {
    if (a.dp <= 32) chunk_t<32>(a, stream);
    else if (a.dp <= 64) chunk_t<64>(a, stream);
    else if (a.dp <= 128) chunk_t<128>(a, stream);
    else chunk_t<256>(a, stream);
}

}  // namespace astrai_mix
