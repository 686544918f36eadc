// Causal sliding-window attention of a block of new tokens (prompt, whole or in portions): bf16
// MFMAs, fp32 scores, weights and sums, output gate in the epilogue. Two kinds of heads:
//   latent        each head has its own keys and values, plus one rotated key part shared by all
//                 heads; a gate per head
//   grouped-query (GQA) `group` heads share keys and values; soft-capped scores, a sink (one more term
//                 exp(0) in the softmax denominator: the running maximum starts at 0 and the sum at
//                 1), a gate per element, each optional
//
// One workgroup per (sequence, head, 128 query tokens), wave r taking 32 of them; key tiles of 32,
// only those some query of the wave can see:
//   S^T = K.Q^T on v_mfma_f32_32x32x16_bf16 with keys as rows and queries as columns, so a lane
//     owns one query (column lane % 32) and 16 scores of a tile: row maxima and sums are per-lane
//     reductions plus one exchange with lane ^ 32;
//   O^T += V^T.P^T with the same instruction: the S^T accumulator is P^T's operand layout already
//     (its register order fixes which keys a lane half contributes), and V^T comes out of the
//     row-major value tile through transposing LDS reads. The weights enter as two bf16 terms,
//     so they keep 16 bits of mantissa.
// A key has two parts in two places, the head's unrotated part and the cache's rotated part; each
// has its own LDS rows. Keys arrive by direct-to-LDS loads in a ring of four tiles, values in two
// 64-key buffers, both one 64-key block ahead: no staging registers, one barrier per block. The
// LDS rows of 16-byte chunks are XOR-swizzled so that the 16 rows an operand read touches (keys) or
// the four rows a transposing read touches (values) fall into different banks. The loads' buffer
// descriptor is rebuilt per block to end at the newest visible key: rows past it and padding
// columns arrive as zeros without predicates.
// A wave's stream is a software pipeline over tiles: the score MFMAs of tile T + 1 are issued among the
// exponentials of tile T, the value MFMAs of tile T among the masking of tile T + 1. One copy of the
// step masks every tile: a second copy without masking costs more in registers and code than the
// compares (157 us against 107 us for 32 x 512 tokens, 16 heads of 128 + 64).
#include "mix_common.cuh"
#include "mix_launchers.h"

namespace astrai_mix {

namespace {

constexpr int kQB = 128;   // query tokens per workgroup
constexpr int kKB = 64;    // keys per block (two tiles)

__device__ __forceinline__ void lds_dma16(__amdgpu_buffer_rsrc_t r, uint8_t* lds_wave_base, uint32_t voff) {
    __builtin_amdgcn_raw_ptr_buffer_load_lds(r, (__attribute__((address_space(3))) void*)lds_wave_base, 16, voff, 0, 0, 0);
}

// which of a row's C chunks sits at position 0: 16 consecutive rows cover all banks
template <int C>
__device__ __forceinline__ int row_swizzle(int row) {
    constexpr int R = C >= 16 ? 1 : 16 / C;   // rows per 256 bytes
    return (row / R) & (C >= 16 ? 15 : C - 1);
}

template <int DN, int DR, int DV, bool GQA>
__global__ __launch_bounds__(256, 2) void mix_prefill_kernel(LatentPrefillArgs a, LatentDims d) {
    constexpr int NKN = DN / 16, NKR = DR / 16, NK = NKN + NKR;   // score MFMA steps
    constexpr int NV = DV / 32;                                   // value column tiles
    constexpr int CN = DN / 8, CR = DR / 8, CV = DV / 8;          // 16-byte chunks per row
    constexpr int kNRow = DN * 2, kRRow = DR * 2, kVRow = DV * 2; // bytes per LDS row
    constexpr int kTile = 32 * (kNRow + kRRow), kRing = 4 * kTile, kVBuf = kKB * kVRow;
    constexpr int JN = CN / 4, JR = CR / 4, JV = CV / 4;          // loads per wave and 64-key block
    constexpr int IN = CN / 2, IR = CR / 2;                       // loads per 32-key tile, all waves
    extern __shared__ __attribute__((aligned(1024))) uint8_t lds[];

    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int qi = lane & 31, h2 = lane >> 5;
    const int groups = a.batch * d.heads;
    const int nqb = (a.seq + kQB - 1) / kQB;
    const int qb = nqb - 1 - (int)(blockIdx.x / groups), bh = (int)(blockIdx.x % groups);   // longest key ranges first
    const int b = bh / d.heads, head = bh % d.heads;
    const int kv_head = GQA ? head / a.group : head, kv_heads = GQA ? d.heads / a.group : d.heads;
    const int dk = d.dn + d.dr;
    const int q0 = qb * kQB;

    const int s_row = q0 + wave * 32 + qi;
    const int64_t tok = (int64_t)b * a.seq + min(s_row, a.seq - 1);
    const int pq = a.start + min(s_row, a.seq - 1), plo = max(pq - d.window + 1, 0);
    // keys of the workgroup, key tiles of the wave (none past the end of the block)
    const int kmax = a.start + min(q0 + kQB, a.seq) - 1;
    const int kmin = max(a.start + q0 - d.window + 1, 0);
    const bool w_live = q0 + wave * 32 < a.seq;
    const int w_first = a.start + q0 + wave * 32, w_last = min(w_first + 31, kmax);
    const int ta = w_live ? (max(w_first - d.window + 1, 0) - kmin) / 32 : 1 << 28;
    const int tb = w_live ? (w_last - kmin) / 32 : -1;
    const int nblocks = (kmax - kmin) / kKB + 1;

    u32x4 qf[NK];
    {
        const uint16_t* q = static_cast<const uint16_t*>(a.proj) + tok * a.ld + head * dk + 8 * h2;
#pragma unroll
        for (int ks = 0; ks < NK; ++ks) {
            const int e = ks < NKN ? ks * 16 : (ks - NKN) * 16;
            const bool ok = ks < NKN ? e < d.dn : e < d.dr;
            qf[ks] = ok ? *reinterpret_cast<const u32x4*>(q + (ks < NKN ? e : d.dn + e)) : u32x4{0, 0, 0, 0};
        }
    }

    const int64_t ldkv = (int64_t)kv_heads * (d.dn + d.vp) * 2, ldc = (d.rp + d.dr) * 2;   // bytes
    const uint8_t* kv = static_cast<const uint8_t*>(a.kv) + ((int64_t)b * a.n_keys - a.key_base) * ldkv +
                        (int64_t)kv_head * (d.dn + d.vp) * 2;
    const uint8_t* kr = static_cast<const uint8_t*>(a.cache) + (int64_t)b * a.max_len * ldc + d.rp * 2;
    // per-lane offsets from a block's first row; a chunk past the real columns asks for nothing
    uint32_t on[JN], orr[DR ? JR : 1], ov[JV];
#pragma unroll
    for (int j = 0; j < JN; ++j) {
        const int row = (wave * JN + j) * (64 / CN) + lane / CN, c = (lane % CN) ^ row_swizzle<CN>(row & 31);
        on[j] = c * 8 < d.dn ? (uint32_t)(row * ldkv) + c * 16 : w8a8::kOutOfRange;
    }
    if constexpr (DR > 0) {
#pragma unroll
        for (int j = 0; j < JR; ++j) {
            const int row = (wave * JR + j) * (64 / CR) + lane / CR, c = (lane % CR) ^ row_swizzle<CR>(row & 31);
            orr[j] = c * 8 < d.dr ? (uint32_t)(row * ldc) + c * 16 : w8a8::kOutOfRange;
        }
    }
    // values: chunk bit 2 (and 3) by the row inside its group of four
    auto v_swizzle = [](int row) { return CV == 16 ? 4 * (row & 3) : 4 * ((row >> 1) & 1); };
#pragma unroll
    for (int j = 0; j < JV; ++j) {
        const int row = (wave * JV + j) * (64 / CV) + lane / CV, c = (lane % CV) ^ v_swizzle(row);
        ov[j] = c * 8 < d.vp ? (uint32_t)(row * ldkv) + c * 16 : w8a8::kOutOfRange;
    }
    auto rows_rsrc = [](const uint8_t* p, int rows, int64_t ld, int bytes) {
        const int64_t n = rows > 0 ? (int64_t)(rows - 1) * ld + bytes : 0;
        return w8a8::make_rsrc(p, (uint32_t)n);
    };
    // tiles t0 and t0 + 1 into their ring slots
    auto dma_k = [&](int t0) {
        const int key = kmin + t0 * 32, rows = min(kmax - key + 1, kKB);
        const __amdgpu_buffer_rsrc_t rn = rows_rsrc(kv + (int64_t)key * ldkv, rows, ldkv, d.dn * 2);
#pragma unroll
        for (int j = 0; j < JN; ++j) {
            const int inst = wave * JN + j;
            lds_dma16(rn, lds + ((t0 + inst / IN) & 3) * kTile + (inst % IN) * 1024, on[j]);
        }
        if constexpr (DR > 0) {
            const __amdgpu_buffer_rsrc_t rr = rows_rsrc(kr + (int64_t)key * ldc, rows, ldc, d.dr * 2);
#pragma unroll
            for (int j = 0; j < JR; ++j) {
                const int inst = wave * JR + j;
                lds_dma16(rr, lds + ((t0 + inst / IR) & 3) * kTile + 32 * kNRow + (inst % IR) * 1024, orr[j]);
            }
        }
    };
    auto dma_v = [&](int kb) {
        const int key = kmin + kb * kKB, rows = min(kmax - key + 1, kKB);
        const __amdgpu_buffer_rsrc_t rv = rows_rsrc(kv + (int64_t)key * ldkv + d.dn * 2, rows, ldkv, d.vp * 2);
#pragma unroll
        for (int j = 0; j < JV; ++j) lds_dma16(rv, lds + kRing + (kb & 1) * kVBuf + (wave * JV + j) * 1024, ov[j]);
    };

    f32x16 o[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int e = 0; e < 16; ++e) o[i][e] = 0.0f;
    // m_run: the maximum the weights are taken against, in log2 units; it follows the running
    // maximum once some query has outgrown it by 2^kSlack (until then weights reach 2^kSlack). It
    // starts far below any score and far above a hidden key's.
    constexpr float kSlack = 8.0f;
    const bool sink = GQA && a.sink;
    float m_run = sink ? 0.0f : 1e-5f * kNegBig, l_run = sink && h2 == 0 ? 1.0f : 0.0f;
    // capped scores leave mask_max4 in log2 units
    const bool capped = GQA && a.softcap > 0.0f;
    const float c = capped ? 1.0f : d.scale * kLog2e;
    const float cap_in = capped ? d.scale / a.softcap : 0.0f, cap_out = a.softcap * kLog2e;
    const f32x16 zero16 = {0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f,
                           0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f};
    // key operand of step ks: chunk (2 ks + h2) ^ swizzle of this lane's row. Rows are powers of two and
    // tiles whole rows, so the step XORs into the whole byte offset: one address register per tile.
    const int kn_lane = qi * kNRow + ((h2 ^ row_swizzle<CN>(qi)) << 4);
    const int kr_lane = 32 * kNRow + qi * kRRow + ((h2 ^ row_swizzle<DR ? CR : CN>(qi)) << 4);
    auto k_frag = [&](int slot, int ks) -> u32x4 {
        const int off = (DR == 0 || ks < NKN) ? ((slot + kn_lane) ^ (ks << 5)) : ((slot + kr_lane) ^ ((ks - NKN) << 5));
        return *reinterpret_cast<const u32x4*>(lds + off);
    };
    // V^T operand of 32 columns x 16 keys: lane half takes rows 4 h2 .. and 8 + 4 h2 .. of the step
    const int v_lane = [&] {
        const int j = (lane & 15) >> 2, q = lane & 3, g1 = (lane >> 4) & 1;
        return (4 * h2 + j) * kVRow + (((2 * g1 + (q >> 1)) ^ v_swizzle(j)) << 4) + ((q & 1) << 3);
    }();
    auto v_frag = [&](int vt, int t, int i) -> u32x4 {
        const uint8_t* src = lds + ((vt + v_lane) ^ (i << 6)) + t * 16 * kVRow;
        return join(lds_read_tr(src), lds_read_tr(src + 8 * kVRow));
    };
    auto mask_max4 = [&](int T, f32x16& s, int g, float m) -> float {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int e = 4 * g + j, key = kmin + T * 32 + g * 8 + h2 * 4 + j;
            if (capped) s[e] = cap_out * tanh_fast(s[e] * cap_in);
            s[e] = (key <= pq && key >= plo) ? s[e] : kNegBig;
            m = fmaxf(m, s[e]);
        }
        return m;
    };
    // In: s_in = masked scores of tile T, m_in their maximum. Out: the values of tile T added to o;
    // s_out = scores of tile T + 1, m_out their maximum. vt: LDS offset of tile T's value rows.
    auto step = [&](int T, f32x16& s_in, float m_in, f32x16& s_out, float& m_out, int vt) {
        const float m_sc = m_in * c;
        if (__any(m_sc > m_run + kSlack)) {
            const float m_new = fmaxf(m_run, m_sc);
            const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
            m_run = m_new;
            l_run *= alpha;
#pragma unroll
            for (int i = 0; i < NV; ++i)
#pragma unroll
                for (int e = 0; e < 16; ++e) o[i][e] *= alpha;
        }
        const int slot = ((T + 1) & 3) * kTile;
        uint32_t hi[8], lo[8];
        float l_add = 0.0f;
        u32x4 kf[NK], vf[2 * NV];
        kf[0] = k_frag(slot, 0);
        kf[1] = k_frag(slot, 1);
#pragma unroll
        for (int ks = 0; ks < NK; ++ks) {
            if (ks + 2 < NK) kf[ks + 2] = k_frag(slot, ks + 2);
            if (ks >= NK - 2) vf[ks - (NK - 2)] = v_frag(vt, 0, ks - (NK - 2));
            s_out = mfma32(kf[ks], qf[ks], ks == 0 ? zero16 : s_out);
#pragma unroll
            for (int p = ks * 8 / NK; p < (ks + 1) * 8 / NK; ++p) {
                const float p0 = __builtin_amdgcn_exp2f(__builtin_fmaf(s_in[2 * p], c, -m_run));
                const float p1 = __builtin_amdgcn_exp2f(__builtin_fmaf(s_in[2 * p + 1], c, -m_run));
                l_add += p0 + p1;
                split2(p0, p1, hi[p], lo[p]);
            }
            }
        l_run += l_add;
        float m = kNegBig;
#pragma unroll
        for (int i = 0; i < 2 * NV; ++i) {
            const int t = i / NV, dt = i % NV;
            if (i + 2 < 2 * NV) vf[i + 2] = v_frag(vt, (i + 2) / NV, (i + 2) % NV);
            const u32x4 ph = {hi[4 * t], hi[4 * t + 1], hi[4 * t + 2], hi[4 * t + 3]};
            const u32x4 pl = {lo[4 * t], lo[4 * t + 1], lo[4 * t + 2], lo[4 * t + 3]};
            o[dt] = mfma32(vf[i], ph, o[dt]);
            o[dt] = mfma32(vf[i], pl, o[dt]);
#pragma unroll
            for (int g = i * 4 / (2 * NV); g < (i + 1) * 4 / (2 * NV); ++g) m = mask_max4(T + 1, s_out, g, m);
            }
        m_out = fmaxf(m, __shfl_xor(m, 32, kWave));
    };
    dma_k(0);
    dma_k(1);
    dma_v(0);
    __builtin_amdgcn_s_waitcnt(0x0070);  // vmcnt(0) lgkmcnt(0)
    __syncthreads();
    f32x16 sa, sb;
    float ma = kNegBig, mb = kNegBig;
#pragma unroll
    for (int e = 0; e < 16; ++e) sa[e] = sb[e] = kNegBig;
    if (ta == 0) {
#pragma unroll
        for (int ks = 0; ks < NK; ++ks) sa = mfma32(k_frag(0, ks), qf[ks], ks == 0 ? zero16 : sa);
        float m = kNegBig;
#pragma unroll
        for (int g = 0; g < 4; ++g) m = mask_max4(0, sa, g, m);
        ma = fmaxf(m, __shfl_xor(m, 32, kWave));
    }
    __syncthreads();  // tile 0's ring slot is overwritten by the first block's loads
    for (int kb = 0; kb < nblocks; ++kb) {
        dma_k(2 * kb + 3);  // tiles 2kb+3, 2kb+4: their ring slots held tiles 2kb-1 and 2kb
        if (kb + 1 < nblocks) dma_v(kb + 1);
        const int vt = kRing + (kb & 1) * kVBuf;
        // (the step before the wave's first tile runs on hidden scores and brings in that tile's)
        if (2 * kb >= ta - 1 && 2 * kb <= tb) step(2 * kb, sa, ma, sb, mb, vt);
        if (2 * kb + 1 >= ta - 1 && 2 * kb + 1 <= tb) step(2 * kb + 1, sb, mb, sa, ma, vt + 32 * kVRow);
        __builtin_amdgcn_s_waitcnt(0x0070);
        __syncthreads();
    }
    if (!w_live) return;
    // normalise, gate, and write through LDS (idle by now), so that rows leave in whole pieces
    const float l = l_run + __shfl_xor(l_run, 32, kWave);
    const uint16_t* gate = static_cast<const uint16_t*>(a.proj) + tok * a.ld + a.g_off;
    float f = 1.0f / l;
    if constexpr (GQA) gate += head * d.vp;
    else f *= sigmoid(Elem<uint16_t>::get(gate + head));
    uint8_t* const mine = lds + wave * 32 * kVRow;
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int g = 0; g < 4; ++g) {
            const int chunk = (4 * i + g) ^ (qi & (CV - 1));
            f32x4 v = {o[i][4 * g] * f, o[i][4 * g + 1] * f, o[i][4 * g + 2] * f, o[i][4 * g + 3] * f};
            if constexpr (GQA) {
                const int col = 32 * i + 8 * g + 4 * h2;
                if (a.g_off >= 0 && col < d.vp) {
                    const f32x4 z = Elem<uint16_t>::get4(gate + col);
#pragma unroll
                    for (int e = 0; e < 4; ++e) v[e] *= sigmoid_fast(z[e]);
                }
            }
            Elem<uint16_t>::put4(reinterpret_cast<uint16_t*>(mine + qi * kVRow + chunk * 16 + h2 * 8), v);
        }
    uint16_t* const out = static_cast<uint16_t*>(a.out) + (((int64_t)b * a.seq + q0 + wave * 32) * d.heads + head) * d.vp;
#pragma unroll
    for (int i = 0; i < CV / 2; ++i) {
        const int row = i * (64 / CV) + lane / CV, ch = lane % CV;
        const u32x4 v = *reinterpret_cast<const u32x4*>(mine + row * kVRow + ((ch ^ (row & (CV - 1))) << 4));
        if (q0 + wave * 32 + row < a.seq && ch * 8 < d.vp)
            *reinterpret_cast<u32x4*>(out + (int64_t)row * d.heads * d.vp + ch * 8) = v;
    }
}

template <int DN, int DR, int DV, bool GQA>
void prefill_t(const LatentPrefillArgs& a, const LatentDims& d, hipStream_t stream) {
    constexpr int shared = 4 * 32 * (DN + DR) * 2 + 2 * kKB * DV * 2;
    static const hipError_t once = hipFuncSetAttribute(reinterpret_cast<const void*>(&mix_prefill_kernel<DN, DR, DV, GQA>),
                                                       hipFuncAttributeMaxDynamicSharedMemorySize, shared);
    (void)once;
    const unsigned blocks = (unsigned)(((a.seq + kQB - 1) / kQB) * a.batch * d.heads);
    mix_prefill_kernel<DN, DR, DV, GQA><<<blocks, 256, shared, stream>>>(a, d);
}

template <int DN, int DR, bool GQA>
void prefill_v(const LatentPrefillArgs& a, const LatentDims& d, hipStream_t stream) {
    if (d.vp <= 64) prefill_t<DN, DR, 64, GQA>(a, d, stream);
    else prefill_t<DN, DR, 128, GQA>(a, d, stream);
}

template <int DN>
void prefill_r(const LatentPrefillArgs& a, const LatentDims& d, hipStream_t stream) {
    if (d.dr <= 32) prefill_v<DN, 32, false>(a, d, stream);
    else prefill_v<DN, 64, false>(a, d, stream);
}

}  // namespace

// (a scale below 1e-4 would bring a hidden key's stand-in within reach of the starting maximum)
bool latent_prefill_supported(const LatentDims& d) {
    return d.dn <= 128 && d.dr <= 64 && d.vp <= 128 && d.scale >= 1e-4f && d.scale <= 1e4f &&
           (int64_t)kKB * d.heads * (d.dn + d.vp) * 2 < (1 << 30);
}

bool launch_latent_prefill(const LatentPrefillArgs& a, const LatentDims& d, hipStream_t stream) {
    if (!latent_prefill_supported(d)) return false;
    if (d.dn <= 64) prefill_r<64>(a, d, stream);
    else prefill_r<128>(a, d, stream);
    return true;
}

bool gqa_prefill_supported(const LatentDims& d) { return d.dr == 0 && latent_prefill_supported(d); }

bool launch_gqa_prefill(const LatentPrefillArgs& a, const LatentDims& d, hipStream_t stream) {
    if (!gqa_prefill_supported(d)) return false;
    if (d.dn <= 64) prefill_v<64, 0, true>(a, d, stream);
    else prefill_v<128, 0, true>(a, d, stream);
    return true;
}

}  // namespace astrai_mix
