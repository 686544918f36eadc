// Causal sliding-window attention of a block of new tokens (prompt, whole or in portions) for
// heads with their own keys and values plus one rotated key part shared by all heads: bf16
// MFMAs, fp32 scores, weights and sums, per-head output gate in the epilogue.
//
// One workgroup per (sequence, head, 128 query tokens), wave r taking 32 of them. Keys in tiles
// of 64, only those some query of the workgroup can see:
//   S^T = K.Q^T on v_mfma_f32_32x32x16_bf16 with keys as rows and queries as columns, so a lane
//     owns one query (column lane % 32) and 16 scores of each half tile: row maxima and sums are
//     per-lane reductions plus one exchange with lane ^ 32;
//   O^T += V^T.P^T with the same instruction: the S^T accumulator is P^T's operand layout already
//     (its register order fixes which keys a lane half contributes), and V^T comes out of the
//     row-major value tile through transposing LDS reads. The weights enter as two bf16 terms,
//     so they keep 16 bits of mantissa.
// A key row is gathered from two places, the head's unrotated part and the cache's rotated part.
// The next tile travels in registers while the current one is multiplied; rows are padded in LDS
// so that operand reads of neighbouring rows fall into different banks. Two workgroups share a
// CU and cover each other's barriers.
#include "mix_common.cuh"
#include "mix_launchers.h"

namespace astrai_mix {

namespace {

constexpr int kQB = 128;   // query tokens per workgroup
constexpr int kKB = 64;    // keys per tile

template <int DK, int DV>
__global__ __launch_bounds__(256, 2) void latent_prefill_kernel(LatentPrefillArgs a, LatentDims d) {
    constexpr int NK = DK / 16;                  // score MFMA steps
    constexpr int NV = DV / 32;                  // value column tiles
    constexpr int kKRow = DK * 2 + 16;           // bytes per key row in LDS
    // value rows: four consecutive rows must cover 256 bytes of banks, 64 apiece
    constexpr int kVRow = (DV * 2) % 128 == 64 ? DV * 2 : DV * 2 + 64;
    constexpr int KC = DK / 8, VC = DV / 8;      // 16-byte chunks per row
    constexpr int NKL = kKB * KC / 256, NVL = kKB * VC / 256;   // loads per thread and tile
    __shared__ __attribute__((aligned(16))) uint8_t lk[kKB * kKRow];
    __shared__ __attribute__((aligned(16))) uint8_t lv[kKB * kVRow];

    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int qi = lane & 31, h2 = lane >> 5;
    const int groups = a.batch * d.heads;
    const int qb = (int)(blockIdx.x / groups), bh = (int)(blockIdx.x % groups);
    const int b = bh / d.heads, head = bh % d.heads;
    const int dk = d.dn + d.dr;
    const int q0 = qb * kQB;

    const int s_row = q0 + wave * 32 + qi;
    const bool live = s_row < a.seq;
    const int64_t tok = (int64_t)b * a.seq + min(s_row, a.seq - 1);
    const int pq = a.start + min(s_row, a.seq - 1);
    const int plo = max(pq - d.window + 1, 0);
    // keys the workgroup / the wave needs
    const int kmax = a.start + min(q0 + kQB, a.seq) - 1;
    const int kmin = max(a.start + q0 - d.window + 1, 0);
    const int w_first = a.start + min(q0 + wave * 32, a.seq - 1), w_last = a.start + min(q0 + wave * 32 + 31, a.seq - 1);
    const bool w_live = q0 + wave * 32 < a.seq;

    u32x4 qf[NK];
    {
        const uint16_t* q = static_cast<const uint16_t*>(a.proj) + tok * a.ld + head * dk + 8 * h2;
#pragma unroll
        for (int ks = 0; ks < NK; ++ks)
            qf[ks] = ks * 16 < dk ? *reinterpret_cast<const u32x4*>(q + ks * 16) : u32x4{0, 0, 0, 0};
    }

    const int64_t ldkv = (int64_t)d.heads * (d.dn + d.vp), ldc = d.rp + d.dr;
    const uint16_t* kv = static_cast<const uint16_t*>(a.kv) + (int64_t)b * a.n_keys * ldkv + (int64_t)head * (d.dn + d.vp);
    const uint16_t* kr = static_cast<const uint16_t*>(a.cache) + (int64_t)b * a.max_len * ldc + d.rp - d.dn;
    u32x4 rk[NKL], rv[NVL];
    auto fetch = [&](int k0) {
#pragma unroll
        for (int i = 0; i < NKL; ++i) {
            const int c = tid + i * 256, row = c / KC, e = (c % KC) * 8;
            const int key = k0 + row;
            const bool ok = key <= kmax && e < dk;
            const uint16_t* p = e < d.dn ? kv + (int64_t)(key - a.key_base) * ldkv : kr + (int64_t)key * ldc;
            rk[i] = ok ? *reinterpret_cast<const u32x4*>(p + e) : u32x4{0, 0, 0, 0};
        }
#pragma unroll
        for (int i = 0; i < NVL; ++i) {
            const int c = tid + i * 256, row = c / VC, e = (c % VC) * 8;
            const int key = k0 + row;
            const bool ok = key <= kmax && e < d.vp;
            rv[i] = ok ? *reinterpret_cast<const u32x4*>(kv + (int64_t)(key - a.key_base) * ldkv + d.dn + e)
                       : u32x4{0, 0, 0, 0};
        }
    };

    f32x16 o[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int e = 0; e < 16; ++e) o[i][e] = 0.0f;
    // m_run: the maximum the weights are taken against, in log2 units; it follows the running
    // maximum once some query has outgrown it by 2^kSlack (until then weights reach 2^kSlack)
    constexpr float kSlack = 8.0f;
    float m_run = 1e-5f * kNegBig, l_run = 0.0f;   // far below any score, far above a hidden key's
    const float c = d.scale * kLog2e;
    const uint8_t* k_src = lk + qi * kKRow + h2 * 16;
    // V^T operand: lane half takes rows 4 h2 .. and 8 + 4 h2 .. of a 16-key step
    const uint8_t* v_src = lv + (4 * h2 + ((lane & 15) >> 2)) * kVRow + ((lane >> 4) & 1) * 32 + (lane & 3) * 8;

    fetch(kmin);
    for (int k0 = kmin; k0 <= kmax; k0 += kKB) {
        __syncthreads();   // every wave is done with the previous tile
#pragma unroll
        for (int i = 0; i < NKL; ++i) {
            const int cc = tid + i * 256;
            *reinterpret_cast<u32x4*>(lk + (cc / KC) * kKRow + (cc % KC) * 16) = rk[i];
        }
#pragma unroll
        for (int i = 0; i < NVL; ++i) {
            const int cc = tid + i * 256;
            *reinterpret_cast<u32x4*>(lv + (cc / VC) * kVRow + (cc % VC) * 16) = rv[i];
        }
        __syncthreads();
        fetch(k0 + kKB);
        // (wave-uniform) does any query of the wave see a key of this tile
        if (!w_live || k0 > w_last || k0 + kKB - 1 < w_first - d.window + 1) continue;
        const bool whole = k0 + kKB - 1 <= w_first && k0 > w_last - d.window;

        f32x16 s[2];
#pragma unroll
        for (int t = 0; t < 2; ++t) {
#pragma unroll
            for (int e = 0; e < 16; ++e) s[t][e] = 0.0f;
#pragma unroll
            for (int ks = 0; ks < NK; ++ks)
                s[t] = mfma32(*reinterpret_cast<const u32x4*>(k_src + t * 32 * kKRow + ks * 32), qf[ks], s[t]);
        }
        float m = kNegBig;
        if (whole) {
#pragma unroll
            for (int t = 0; t < 2; ++t)
#pragma unroll
                for (int e = 0; e < 16; ++e) {
                    s[t][e] *= c;
                    m = fmaxf(m, s[t][e]);
                }
        } else {
#pragma unroll
            for (int t = 0; t < 2; ++t)
#pragma unroll
                for (int e = 0; e < 16; ++e) {
                    const int key = k0 + t * 32 + (e >> 2) * 8 + h2 * 4 + (e & 3);
                    s[t][e] = (key <= pq && key >= plo) ? s[t][e] * c : kNegBig;
                    m = fmaxf(m, s[t][e]);
                }
        }
        m = fmaxf(m, __shfl_xor(m, 32, kWave));
        if (__any(m > m_run + kSlack)) {
            const float m_new = fmaxf(m_run, m);
            const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
            m_run = m_new;
            l_run *= alpha;
#pragma unroll
            for (int i = 0; i < NV; ++i)
#pragma unroll
                for (int e = 0; e < 16; ++e) o[i][e] *= alpha;
        }
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                u32x4 hi, lo;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const float p0 = __builtin_amdgcn_exp2f(s[t][8 * u + 2 * e] - m_run);
                    const float p1 = __builtin_amdgcn_exp2f(s[t][8 * u + 2 * e + 1] - m_run);
                    l_run += p0 + p1;
                    uint32_t a2, b2;
                    split2(p0, p1, a2, b2);
                    hi[e] = a2;
                    lo[e] = b2;
                }
                const uint8_t* v = v_src + (t * 32 + u * 16) * kVRow;
#pragma unroll
                for (int i = 0; i < NV; ++i) {
                    const u32x4 vf = join(lds_read_tr(v + i * 64), lds_read_tr(v + i * 64 + 8 * kVRow));
                    o[i] = mfma32(vf, hi, o[i]);
                    o[i] = mfma32(vf, lo, o[i]);
                }
            }
    }
    if (!live) return;
    const float l = l_run + __shfl_xor(l_run, 32, kWave);
    const float gate = sigmoid(Elem<uint16_t>::get(static_cast<const uint16_t*>(a.proj) + tok * a.ld + a.g_off + head));
    const float f = gate / l;
    uint16_t* out = static_cast<uint16_t*>(a.out) + (tok * d.heads + head) * d.vp;
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int e4 = 0; e4 < 4; ++e4) {
            const int v = i * 32 + e4 * 8 + h2 * 4;
            if (v < d.vp)
                Elem<uint16_t>::put4(out + v, f32x4{o[i][4 * e4] * f, o[i][4 * e4 + 1] * f, o[i][4 * e4 + 2] * f,
                                                    o[i][4 * e4 + 3] * f});
        }
}

template <int DK, int DV>
void prefill_t(const LatentPrefillArgs& a, const LatentDims& d, hipStream_t stream) {
    const unsigned blocks = (unsigned)(((a.seq + kQB - 1) / kQB) * a.batch * d.heads);
    latent_prefill_kernel<DK, DV><<<blocks, 256, 0, stream>>>(a, d);
}

template <int DK>
void prefill_k(const LatentPrefillArgs& a, const LatentDims& d, hipStream_t stream) {
    if (d.vp <= 64) prefill_t<DK, 64>(a, d, stream);
    else prefill_t<DK, 128>(a, d, stream);
}

}  // namespace

bool latent_prefill_supported(const LatentDims& d) { return d.dn + d.dr <= 256 && d.vp <= 128; }

bool launch_latent_prefill(const LatentPrefillArgs& a, const LatentDims& d, hipStream_t stream) {
    if (!latent_prefill_supported(d)) return false;
    const int dk = d.dn + d.dr;
    if (dk <= 64) prefill_k<64>(a, d, stream);
    else if (dk <= 96) prefill_k<96>(a, d, stream);
    else if (dk <= 128) prefill_k<128>(a, d, stream);
    else if (dk <= 160) prefill_k<160>(a, d, stream);
    else if (dk <= 192) prefill_k<192>(a, d, stream);
    else prefill_k<256>(a, d, stream);
    return true;
}

}  // namespace astrai_mix
