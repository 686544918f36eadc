// extern "C" entry points of libastrai_mix.so (declared in include/astrai_mix.h): argument
// validation and launch check. Nothing here allocates, frees or synchronises.
#include "../../include/astrai_mix.h"

#include <hip/hip_runtime.h>

#include <cstdarg>
#include <cstdio>

#include "mix_launchers.h"

static_assert(astrai_mix::kMaxSplit == ASTRAI_MIX_MAX_SPLIT && astrai_mix::kLightningChunk == ASTRAI_MIX_LIGHTNING_CHUNK);

namespace {

using namespace astrai_mix;

thread_local char g_err[256] = "";

int fail(int code, const char* fmt, ...) {
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(g_err, sizeof(g_err), fmt, ap);
    va_end(ap);
    return code;
}

int check_launch(const char* what) {
    const hipError_t e = hipGetLastError();
    if (e != hipSuccess) return fail(ASTRAI_MIX_LAUNCH_FAILED, "%s: %s", what, hipGetErrorString(e));
    return ASTRAI_MIX_OK;
}

template <typename... P>
int check_ptrs(const char* what, P... p) {
    const void* all[] = {p...};
    for (const void* q : all) {
        if (!q) return fail(ASTRAI_MIX_BAD_ARG, "%s: null pointer", what);
        if (reinterpret_cast<uintptr_t>(q) & 15u)
            return fail(ASTRAI_MIX_BAD_ARG, "%s: pointers must be 16-byte aligned", what);
    }
    return ASTRAI_MIX_OK;
}

int check_dtype(const char* what, int dtype) {
    if (dtype != ASTRAI_MIX_BF16 && dtype != ASTRAI_MIX_F32)
        return fail(ASTRAI_MIX_BAD_ARG, "%s: dtype must be 0 (bf16) or 1 (float)", what);
    return ASTRAI_MIX_OK;
}

constexpr int64_t kMaxInt = 0x7fffffff, kMaxGridYZ = 65535;

bool pad32(int64_t v, int64_t lo) { return v >= lo && v % 32 == 0 && v <= (1 << 20); }

int check_heads(const char* what, int64_t heads, int64_t dn, int64_t dr, int64_t rp, int64_t vp) {
    if (heads <= 0 || heads > kMaxGridYZ || !pad32(dn, 0) || !pad32(dr, 0) || dn + dr == 0 || !pad32(rp, 32) ||
        !pad32(vp, 32) || heads * (dn + dr) > kMaxInt || heads * (dn + vp) > kMaxInt)
        return fail(ASTRAI_MIX_BAD_ARG, "%s: head sizes must be positive multiples of 32 (heads %lld, dn %lld, dr %lld, "
                    "rp %lld, vp %lld)", what, (long long)heads, (long long)dn, (long long)dr, (long long)rp, (long long)vp);
    return ASTRAI_MIX_OK;
}

int check_block(const char* what, int64_t batch, int64_t seq, int64_t max_len, int64_t ld, int64_t need) {
    if (batch <= 0 || seq <= 0 || max_len < seq || max_len > (1 << 30) || batch > kMaxGridYZ || batch * seq > kMaxInt)
        return fail(ASTRAI_MIX_BAD_ARG, "%s: bad batch %lld, seq %lld, max_len %lld", what, (long long)batch,
                    (long long)seq, (long long)max_len);
    if (ld % 8 != 0 || ld < need || ld > kMaxInt)
        return fail(ASTRAI_MIX_BAD_ARG, "%s: row stride %lld (need a multiple of 8, at least %lld)", what, (long long)ld,
                    (long long)need);
    return ASTRAI_MIX_OK;
}

int window_of(int64_t window) { return (int)(window > (1 << 30) ? (1 << 30) : window); }

LatentDims dims(int64_t heads, int64_t dn, int64_t dr, int64_t rp, int64_t vp, int64_t window, float scale) {
    LatentDims d;
    d.heads = (int)heads;
    d.dn = (int)dn;
    d.dr = (int)dr;
    d.rp = (int)rp;
    d.vp = (int)vp;
    d.window = window_of(window);
    d.scale = scale;
    return d;
}

int check_lightning(const char* what, int64_t ld, int64_t q_off, int64_t k_off, int64_t v_off, int64_t batch, int64_t seq,
                    int64_t heads, int64_t dp, int64_t vp) {
    if (heads <= 0 || !pad32(dp, 32) || !pad32(vp, 32))
        return fail(ASTRAI_MIX_BAD_ARG, "%s: head sizes must be positive multiples of 32 (heads %lld, dp %lld, vp %lld)",
                    what, (long long)heads, (long long)dp, (long long)vp);
    if (batch <= 0 || seq <= 0 || batch * heads > kMaxGridYZ || batch * seq > kMaxInt)
        return fail(ASTRAI_MIX_BAD_ARG, "%s: bad batch %lld, seq %lld (batch * heads <= 65535)", what, (long long)batch,
                    (long long)seq);
    if (ld % 8 || q_off % 8 || k_off % 8 || v_off % 8 || q_off < 0 || k_off < 0 || v_off < 0 || ld > kMaxInt ||
        q_off + heads * dp > ld || k_off + heads * dp > ld || v_off + heads * vp > ld)
        return fail(ASTRAI_MIX_BAD_ARG, "%s: projection columns do not fit a row of %lld", what, (long long)ld);
    return ASTRAI_MIX_OK;
}

LightningArgs lightning_args(const void* proj, int64_t ld, int64_t q_off, int64_t k_off, int64_t v_off,
                             const float* decay_pow, float* state, float* seg_state, void* out, int64_t batch, int64_t seq,
                             int64_t heads, int64_t dp, int64_t vp, int64_t nseg) {
    LightningArgs a;
    a.proj = proj;
    a.ld = ld;
    a.q_off = (int)q_off;
    a.k_off = (int)k_off;
    a.v_off = (int)v_off;
    a.decay_pow = decay_pow;
    a.state = state;
    a.seg_state = seg_state;
    a.out = out;
    a.batch = (int)batch;
    a.seq = (int)seq;
    a.heads = (int)heads;
    a.dp = (int)dp;
    a.vp = (int)vp;
    a.nseg = (int)nseg;
    return a;
}

}  // namespace

#define MIX_TRY(expr)                     \
    do {                                  \
        const int rc_ = (expr);           \
        if (rc_ != ASTRAI_MIX_OK) return rc_; \
    } while (0)

extern "C" {

int astrai_mix_abi_version(void) { return ASTRAI_MIX_ABI_VERSION; }

const char* astrai_mix_last_error(void) { return g_err; }

int astrai_mix_residual_norm(const void* y, const float* x_in, float* x_out, const float* w_post, const float* w_pre,
                             void* h, int64_t rows, int64_t width, float mult, float eps, int dtype, void* stream) {
    MIX_TRY(check_dtype("residual_norm", dtype));
    MIX_TRY(check_ptrs("residual_norm", y, (const void*)x_in, (const void*)x_out, (const void*)w_post,
                       (const void*)w_pre, (const void*)h));
    if (rows < 0 || rows > kMaxInt || width <= 0 || width > (1 << 24))
        return fail(ASTRAI_MIX_BAD_ARG, "residual_norm: bad size %lld x %lld", (long long)rows, (long long)width);
    if (rows == 0) return ASTRAI_MIX_OK;
    ResidualNormArgs a = {y, nullptr, x_in, x_out, w_post, w_pre, h, rows, 0, (int)width, mult, eps};
    launch_residual_norm(a, dtype, static_cast<hipStream_t>(stream));
    return check_launch("residual_norm");
}

int astrai_mix_embed_norm(const void* table, const int64_t* tokens, float* x_out, const float* w_pre, void* h,
                          int64_t rows, int64_t width, int64_t vocab, float eps, int dtype, void* stream) {
    MIX_TRY(check_dtype("embed_norm", dtype));
    if (!tokens) return fail(ASTRAI_MIX_BAD_ARG, "embed_norm: null pointer");
    MIX_TRY(check_ptrs("embed_norm", table, (const void*)x_out, (const void*)w_pre, (const void*)h));
    if (rows < 0 || rows > kMaxInt || width <= 0 || width > (1 << 24) || vocab <= 0)
        return fail(ASTRAI_MIX_BAD_ARG, "embed_norm: bad size %lld x %lld, vocab %lld", (long long)rows, (long long)width,
                    (long long)vocab);
    if (rows == 0) return ASTRAI_MIX_OK;
    ResidualNormArgs a = {table, tokens, nullptr, x_out, nullptr, w_pre, h, rows, vocab, (int)width, 0.0f, eps};
    launch_residual_norm(a, dtype, static_cast<hipStream_t>(stream));
    return check_launch("embed_norm");
}

int astrai_mix_silu_mul(const void* gu, void* h, int64_t rows, int64_t ff, int dtype, void* stream) {
    MIX_TRY(check_dtype("silu_mul", dtype));
    MIX_TRY(check_ptrs("silu_mul", gu, (const void*)h));
    if (rows < 0 || ff <= 0 || ff % 8 || ff > (1 << 24))
        return fail(ASTRAI_MIX_BAD_ARG, "silu_mul: bad size %lld x %lld", (long long)rows, (long long)ff);
    if (rows == 0) return ASTRAI_MIX_OK;
    launch_silu_mul(gu, h, rows, (int)ff, dtype, static_cast<hipStream_t>(stream));
    return check_launch("silu_mul");
}

int astrai_mix_gated_rms_norm(const void* o, const void* g, int64_t ldg, const float* w, void* out, int64_t rows,
                              int64_t n, int64_t count, float eps, int dtype, void* stream) {
    MIX_TRY(check_dtype("gated_rms_norm", dtype));
    MIX_TRY(check_ptrs("gated_rms_norm", o, g, (const void*)w, (const void*)out));
    if (rows < 0 || rows > kMaxInt || n <= 0 || n % 4 || n > (1 << 24) || ldg % 4 || ldg < n || count <= 0 || count > n)
        return fail(ASTRAI_MIX_BAD_ARG, "gated_rms_norm: bad size %lld x %lld (%lld counted, stride %lld)",
                    (long long)rows, (long long)n, (long long)count, (long long)ldg);
    if (rows == 0) return ASTRAI_MIX_OK;
    launch_gated_rms_norm(o, g, ldg, w, out, rows, (int)n, (int)count, eps, dtype, static_cast<hipStream_t>(stream));
    return check_launch("gated_rms_norm");
}

int astrai_mix_latent_append(void* proj, int64_t ld, int64_t dkv_off, const float* rot, int64_t rot_rows, int64_t half,
                             const int64_t* positions, const float* norm_w, void* cache, const void* w_uk_t, void* q_abs,
                             int64_t batch, int64_t seq, int64_t max_len, int64_t heads, int64_t dn, int64_t dr, int64_t rp, int64_t kv_rank,
                             float eps, int dtype, void* stream) {
    MIX_TRY(check_dtype("latent_append", dtype));
    MIX_TRY(check_ptrs("latent_append", (const void*)proj, (const void*)rot));
    if (!positions) return fail(ASTRAI_MIX_BAD_ARG, "latent_append: null pointer");
    if (dkv_off >= 0) MIX_TRY(check_ptrs("latent_append", (const void*)norm_w, (const void*)cache));
    MIX_TRY(check_heads("latent_append", heads, dn, dr, rp, 32));
    MIX_TRY(check_block("latent_append", batch, seq, max_len, ld,
                        dkv_off >= 0 ? dkv_off + rp + dr : heads * (dn + dr)));
    if ((dkv_off >= 0 && (dkv_off % 8 || dkv_off < heads * (dn + dr))) || half <= 0 || 2 * half > dr || kv_rank <= 0 ||
        kv_rank > rp || rot_rows <= 0 || heads * half > kMaxInt)
        return fail(ASTRAI_MIX_BAD_ARG, "latent_append: bad columns (dkv_off %lld, half %lld, kv_rank %lld)",
                    (long long)dkv_off, (long long)half, (long long)kv_rank);
    if (q_abs) {
        MIX_TRY(check_ptrs("latent_append", w_uk_t, (const void*)q_abs));
        if (dtype != ASTRAI_MIX_BF16 || batch * seq > (1 << 20) || heads * (rp / 32) > (1 << 20) ||
            batch * seq * heads * ((rp + 63) / 64) > kMaxInt)
            return fail(ASTRAI_MIX_UNSUPPORTED, "latent_append: absorbed queries are bf16, for %lld tokens at most", 1LL << 20);
    }
    LatentAppendArgs a;
    a.proj = proj;
    a.ld = ld;
    a.dkv_off = (int)dkv_off;
    a.rot = rot;
    a.positions = positions;
    a.norm_w = norm_w;
    a.cache = cache;
    a.w_uk_t = w_uk_t;
    a.q_abs = q_abs;
    a.tokens = batch * seq;
    a.rot_rows = rot_rows;
    a.seq = (int)seq;
    a.max_len = (int)max_len;
    a.half = (int)half;
    a.kv_rank = (int)kv_rank;
    a.eps = eps;
    launch_latent_append(a, dims(heads, dn, dr, rp, 32, 1, 1.0f), dtype, static_cast<hipStream_t>(stream));
    return check_launch("latent_append");
}

int astrai_mix_latent_prefill(const void* proj, int64_t ld, int64_t g_off, const void* kv, const void* cache, void* out,
                              int64_t batch, int64_t seq, int64_t max_len, int64_t start, int64_t key_base,
                              int64_t n_keys, int64_t heads, int64_t dn, int64_t dr, int64_t rp, int64_t vp,
                              int64_t window, float scale, void* stream) {
    MIX_TRY(check_ptrs("latent_prefill", proj, kv, cache, (const void*)out));
    MIX_TRY(check_heads("latent_prefill", heads, dn, dr, rp, vp));
    MIX_TRY(check_block("latent_prefill", batch, seq, max_len, ld, heads * (dn + dr)));
    const int64_t oldest = start - window + 1 > 0 ? start - window + 1 : 0;
    if (window <= 0 || start < 0 || start + seq > max_len || key_base < 0 || key_base > oldest ||
        key_base + n_keys < start + seq)
        return fail(ASTRAI_MIX_BAD_ARG, "latent_prefill: keys %lld .. %lld do not cover tokens %lld .. %lld with window %lld",
                    (long long)key_base, (long long)(key_base + n_keys - 1), (long long)start, (long long)(start + seq - 1),
                    (long long)window);
    if (g_off < 0 || g_off + heads > ld) return fail(ASTRAI_MIX_BAD_ARG, "latent_prefill: bad gate column");
    const LatentDims d = dims(heads, dn, dr, rp, vp, window, scale);
    if (!latent_prefill_supported(d) || ((seq + 127) / 128) * batch * heads > kMaxInt)
        return fail(ASTRAI_MIX_UNSUPPORTED, "latent_prefill: head sizes %lld + %lld, value %lld (at most 128, 64, 128) or scale %g",
                    (long long)dn, (long long)dr, (long long)vp, (double)scale);
    LatentPrefillArgs a;
    a.proj = proj;
    a.ld = ld;
    a.g_off = (int)g_off;
    a.kv = kv;
    a.cache = cache;
    a.out = out;
    a.batch = (int)batch;
    a.seq = (int)seq;
    a.max_len = (int)max_len;
    a.start = (int)start;
    a.key_base = (int)key_base;
    a.n_keys = (int)n_keys;
    launch_latent_prefill(a, d, static_cast<hipStream_t>(stream));
    return check_launch("latent_prefill");
}

int64_t astrai_mix_latent_rows_workspace_floats(int64_t tokens, int64_t heads, int64_t rp, int64_t nsplit) {
    return latent_rows_workspace_floats(dims(heads, 32, 32, rp, 32, 1, 1.0f), tokens, (int)nsplit);
}

int astrai_mix_latent_rows(const void* proj, int64_t ld, int64_t g_off, const void* w_ukv, const void* cache,
                           const int64_t* positions, void* q_abs, float* ws, void* out,
                           int64_t batch, int64_t seq, int64_t max_len, int64_t heads, int64_t dn, int64_t dr,
                           int64_t rp, int64_t vp, int64_t window, float scale, int64_t nsplit, void* stream) {
    MIX_TRY(check_ptrs("latent_rows", proj, w_ukv, cache, (const void*)q_abs, (const void*)ws, (const void*)out));
    if (!positions) return fail(ASTRAI_MIX_BAD_ARG, "latent_rows: null pointer");
    MIX_TRY(check_heads("latent_rows", heads, dn, dr, rp, vp));
    MIX_TRY(check_block("latent_rows", batch, seq, max_len, ld, heads * (dn + dr)));
    if (window <= 0 || g_off < 0 || g_off + heads > ld || nsplit < 1 || nsplit > kMaxSplit)
        return fail(ASTRAI_MIX_BAD_ARG, "latent_rows: bad window, gate column or nsplit %lld", (long long)nsplit);
    const LatentDims d = dims(heads, dn, dr, rp, vp, window, scale);
    if (!latent_rows_mfma_supported(d) || seq * heads * nsplit > kMaxInt || (batch * seq + 15) / 16 > kMaxGridYZ ||
        batch * seq * heads > kMaxInt || max_len * (rp + dr) * 2 >= kMaxInt)
        return fail(ASTRAI_MIX_UNSUPPORTED, "latent_rows: latent %lld + %lld (at most 1024, 64), too many rows or a sequence of 2 GiB",
                    (long long)rp, (long long)dr);
    LatentRowsArgs a = {proj, ld, (int)g_off, w_ukv, cache, positions, q_abs, q_abs, ws, out,
                        (int)batch, (int)seq, (int)max_len, (int)nsplit};
    launch_latent_rows_mfma(a, d, static_cast<hipStream_t>(stream));
    return check_launch("latent_rows");
}

int astrai_mix_latent_rows_general(const void* proj, int64_t ld, int64_t g_off, const void* w_ukv, const void* cache,
                                   const int64_t* positions, void* out, int64_t batch, int64_t seq, int64_t max_len,
                                   int64_t heads, int64_t dn, int64_t dr, int64_t rp, int64_t vp, int64_t window,
                                   float scale, int dtype, void* stream) {
    MIX_TRY(check_dtype("latent_rows_general", dtype));
    MIX_TRY(check_ptrs("latent_rows_general", proj, w_ukv, cache, (const void*)out));
    if (!positions) return fail(ASTRAI_MIX_BAD_ARG, "latent_rows_general: null pointer");
    MIX_TRY(check_heads("latent_rows_general", heads, dn, dr, rp, vp));
    MIX_TRY(check_block("latent_rows_general", batch, seq, max_len, ld, heads * (dn + dr)));
    if (window <= 0 || g_off < 0 || g_off + heads > ld)
        return fail(ASTRAI_MIX_BAD_ARG, "latent_rows_general: bad window or gate column");
    const LatentDims d = dims(heads, dn, dr, rp, vp, window, scale);
    if (!latent_rows_general_supported(d))
        return fail(ASTRAI_MIX_UNSUPPORTED, "latent_rows_general: latent %lld, rotated %lld (at most 2048, 512)",
                    (long long)rp, (long long)dr);
    LatentRowsArgs a = {proj, ld, (int)g_off, w_ukv, cache, positions, nullptr, nullptr, nullptr, out,
                        (int)batch, (int)seq, (int)max_len, 1};
    launch_latent_rows_general(a, d, dtype, static_cast<hipStream_t>(stream));
    return check_launch("latent_rows_general");
}

int astrai_mix_lightning_chunk(const void* proj, int64_t ld, int64_t q_off, int64_t k_off, int64_t v_off,
                               const float* decay_pow, float* state, float* seg_state, void* out, int64_t batch,
                               int64_t seq, int64_t heads, int64_t dp, int64_t vp, int64_t nseg, void* stream) {
    MIX_TRY(check_ptrs("lightning_chunk", proj, (const void*)decay_pow, (const void*)state, (const void*)out));
    MIX_TRY(check_lightning("lightning_chunk", ld, q_off, k_off, v_off, batch, seq, heads, dp, vp));
    if (nseg < 1 || nseg > (seq + kLightningChunk - 1) / kLightningChunk || (nseg > 1 && !seg_state))
        return fail(ASTRAI_MIX_BAD_ARG, "lightning_chunk: bad nseg %lld", (long long)nseg);
    if (!lightning_chunk_supported((int)dp, (int)vp))
        return fail(ASTRAI_MIX_UNSUPPORTED, "lightning_chunk: head size %lld (at most 256)", (long long)dp);
    launch_lightning_chunk(lightning_args(proj, ld, q_off, k_off, v_off, decay_pow, state, seg_state, out, batch, seq,
                                          heads, dp, vp, nseg), static_cast<hipStream_t>(stream));
    return check_launch("lightning_chunk");
}

int astrai_mix_lightning_step(const void* proj, int64_t ld, int64_t q_off, int64_t k_off, int64_t v_off,
                              const float* decay_pow, float* state, void* out, int64_t batch, int64_t seq,
                              int64_t heads, int64_t dp, int64_t vp, int dtype, void* stream) {
    MIX_TRY(check_dtype("lightning_step", dtype));
    MIX_TRY(check_ptrs("lightning_step", proj, (const void*)decay_pow, (const void*)state, (const void*)out));
    MIX_TRY(check_lightning("lightning_step", ld, q_off, k_off, v_off, batch, seq, heads, dp, vp));
    if (!lightning_step_supported((int)dp, (int)vp))
        return fail(ASTRAI_MIX_UNSUPPORTED, "lightning_step: head size %lld (at most 1024)", (long long)dp);
    launch_lightning_step(lightning_args(proj, ld, q_off, k_off, v_off, decay_pow, state, nullptr, out, batch, seq,
                                         heads, dp, vp, 1), dtype, static_cast<hipStream_t>(stream));
    return check_launch("lightning_step");
}

}  // extern "C"
