// extern "C" entry points of libastrai_mix.so (declared in include/astrai_mix.h): argument
// validation and launch check. Nothing here allocates, frees or synchronises.
#include "../../include/astrai_mix.h"

#include <hip/hip_runtime.h>

#include <cstdarg>
#include <cstdio>

#include "mix_launchers.h"

static_assert(astrai_mix::kMaxSplit == ASTRAI_MIX_MAX_SPLIT && astrai_mix::kLightningChunk == ASTRAI_MIX_LIGHTNING_CHUNK);
static_assert(astrai_mix::kRingSteps == ASTRAI_MIX_RING_STEPS && astrai_mix::kDeltaChunk == ASTRAI_MIX_DELTA_CHUNK);
static_assert(astrai_mix::kActSilu == ASTRAI_MIX_SILU && astrai_mix::kActGelu == ASTRAI_MIX_GELU);

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

#define MIX_TRY(expr)                     \
    do {                                  \
        const int rc_ = (expr);           \
        if (rc_ != ASTRAI_MIX_OK) return rc_; \
    } while (0)

int check_gqa(const char* what, int64_t heads, int64_t kv_heads, int64_t dk, int64_t vp) {
    if (heads <= 0 || kv_heads <= 0 || heads % kv_heads || heads > kMaxGridYZ || !pad32(dk, 32) || !pad32(vp, 32) ||
        heads * dk > kMaxInt || heads * vp > kMaxInt || kv_heads * (dk + vp) > kMaxInt)
        return fail(ASTRAI_MIX_BAD_ARG, "%s: bad heads %lld / %lld or head sizes %lld, %lld (positive multiples of 32)", what,
                    (long long)heads, (long long)kv_heads, (long long)dk, (long long)vp);
    return ASTRAI_MIX_OK;
}

int check_gate(const char* what, int64_t ld, int64_t g_off, int64_t cols) {
    if (g_off >= 0 && (g_off % 8 || g_off + cols > ld)) return fail(ASTRAI_MIX_BAD_ARG, "%s: bad gate columns", what);
    return ASTRAI_MIX_OK;
}

GqaDims gqa_dims(int64_t heads, int64_t kv_heads, int64_t dk, int64_t vp, int64_t window, float scale, float softcap,
                 int sink) {
    return GqaDims{(int)heads, (int)kv_heads, (int)dk, (int)vp, window_of(window), scale, softcap, sink};
}

int check_conv(const char* what, int64_t ld, int64_t off, int64_t cols, const float* w, const float* bias, int64_t taps,
               const void* ring, const int64_t* positions) {
    MIX_TRY(check_ptrs(what, (const void*)w, ring));
    if (!positions) return fail(ASTRAI_MIX_BAD_ARG, "%s: null pointer", what);
    if (bias) MIX_TRY(check_ptrs(what, (const void*)bias));
    if (taps < 1 || taps > 1024 || cols <= 0 || cols % 4 || off < 0 || off % 4 || off + cols > ld)
        return fail(ASTRAI_MIX_BAD_ARG, "%s: bad columns %lld .. + %lld of %lld or taps %lld", what, (long long)off,
                    (long long)cols, (long long)ld, (long long)taps);
    return ASTRAI_MIX_OK;
}

ConvArgs conv_args(const void* proj, int64_t ld, int64_t off, int64_t cols, const float* w, const float* bias, int64_t taps,
                   void* ring, const int64_t* positions, void* out, int64_t batch, int64_t seq, int silu) {
    return ConvArgs{proj, ld, (int)off, (int)cols, w, bias, ring, positions, out, (int)batch, (int)seq, (int)taps,
                    (int)taps - 1 + kRingSteps, silu};
}

int check_rglru(const char* what, int64_t ld, int64_t y_off, int64_t batch, int64_t seq, int64_t blocks, int64_t bp) {
    MIX_TRY(check_block(what, batch, seq, seq, ld, 8));
    if (blocks <= 0 || !pad32(bp, 32) || blocks * bp > kMaxInt / 64 || y_off < 0 || y_off % 4 || y_off + blocks * bp > ld)
        return fail(ASTRAI_MIX_BAD_ARG, "%s: bad blocks %lld x %lld (a multiple of 32) or columns", what, (long long)blocks,
                    (long long)bp);
    return ASTRAI_MIX_OK;
}

RglruArgs rglru_args(const void* u, const void* proj, int64_t ld, int64_t y_off, const void* w_r,
                     const void* w_i, const float* b_r, const float* b_i, const float* coef, float* state, float* scratch,
                     void* out, int64_t batch, int64_t seq, int64_t blocks, int64_t bp, int64_t nseg) {
    RglruArgs a = {};
    a.proj = proj;
    a.ld = ld;
    a.y_off = (int)y_off;
    a.u = u;
    a.w_r = w_r;
    a.w_i = w_i;
    a.b_r = b_r;
    a.b_i = b_i;
    a.coef = coef;
    a.state = state;
    a.scratch = scratch;
    a.out = out;
    a.batch = (int)batch;
    a.seq = (int)seq;
    a.blocks = (int)blocks;
    a.bp = (int)bp;
    a.nseg = (int)nseg;
    return a;
}

int check_delta(const char* what, int64_t ld, int64_t b_off, int64_t batch, int64_t seq, int64_t heads, int64_t kv_heads,
                int64_t dp, int64_t vp) {
    MIX_TRY(check_gqa(what, heads, kv_heads, dp, vp));
    MIX_TRY(check_block(what, batch, seq, seq, ld, 8));
    if (b_off < 0 || b_off + heads > ld || 2 * kv_heads * dp + heads * vp > kMaxInt)
        return fail(ASTRAI_MIX_BAD_ARG, "%s: bad step-size columns", what);
    return ASTRAI_MIX_OK;
}

}  // namespace

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

int astrai_mix_sum_norm(const void* y, int64_t ldy, const int64_t* tokens, int64_t vocab, float mult, const float* x_in,
                        const void* u, int64_t ldu, const float* vec, float* x_out, const float* w, void* h,
                        int64_t rows, int64_t width, float eps, int y_float, int dtype, void* stream) {
    MIX_TRY(check_dtype("sum_norm", dtype));
    MIX_TRY(check_ptrs("sum_norm", y, (const void*)x_out, (const void*)h));
    if (x_in) MIX_TRY(check_ptrs("sum_norm", (const void*)x_in));
    if (u) MIX_TRY(check_ptrs("sum_norm", u));
    if (vec) MIX_TRY(check_ptrs("sum_norm", (const void*)vec));
    if (w) MIX_TRY(check_ptrs("sum_norm", (const void*)w));
    if (rows < 0 || rows > kMaxInt || width <= 0 || width > (1 << 24) || ldy < width || (u && ldu < width) ||
        (tokens && vocab <= 0))
        return fail(ASTRAI_MIX_BAD_ARG, "sum_norm: bad size %lld x %lld (strides %lld, %lld)", (long long)rows,
                    (long long)width, (long long)ldy, (long long)ldu);
    if (rows == 0) return ASTRAI_MIX_OK;
    const SumNormArgs a = {y, ldy, tokens, x_in, u, u ? ldu : 0, vec, x_out, w, h, rows, vocab, (int)width, mult, eps};
    launch_sum_norm(a, dtype, y_float != 0, static_cast<hipStream_t>(stream));
    return check_launch("sum_norm");
}

int astrai_mix_act_mul(const void* gu, void* h, int64_t rows, int64_t ff, int act, int dtype, void* stream) {
    MIX_TRY(check_dtype("act_mul", dtype));
    MIX_TRY(check_ptrs("act_mul", gu, (const void*)h));
    if (rows < 0 || ff <= 0 || ff % 8 || ff > (1 << 24) || (act != ASTRAI_MIX_SILU && act != ASTRAI_MIX_GELU))
        return fail(ASTRAI_MIX_BAD_ARG, "act_mul: bad size %lld x %lld or activation %d", (long long)rows, (long long)ff, act);
    if (rows == 0) return ASTRAI_MIX_OK;
    launch_act_mul(gu, h, rows, (int)ff, act, dtype, static_cast<hipStream_t>(stream));
    return check_launch("act_mul");
}

int astrai_mix_head_gated_rms_norm(const void* o, const void* g, int64_t ldg, const float* w, void* out, int64_t rows,
                                   int64_t heads, int64_t vp, int64_t count, float eps, int dtype, void* stream) {
    MIX_TRY(check_dtype("head_gated_rms_norm", dtype));
    MIX_TRY(check_ptrs("head_gated_rms_norm", o, g, (const void*)w, (const void*)out));
    if (rows < 0 || heads <= 0 || vp <= 0 || vp % 4 || vp > (1 << 20) || rows * heads > kMaxInt || ldg % 4 ||
        ldg < heads * vp || count <= 0 || count > vp)
        return fail(ASTRAI_MIX_BAD_ARG, "head_gated_rms_norm: bad size %lld x %lld x %lld (%lld counted, stride %lld)",
                    (long long)rows, (long long)heads, (long long)vp, (long long)count, (long long)ldg);
    if (rows == 0) return ASTRAI_MIX_OK;
    const HeadNormArgs a = {o, g, ldg, w, out, rows, (int)heads, (int)vp, (int)count, eps};
    launch_head_gated_rms_norm(a, dtype, static_cast<hipStream_t>(stream));
    return check_launch("head_gated_rms_norm");
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

int astrai_mix_gqa_append(void* proj, int64_t ld, int64_t k_off, int64_t v_off, const float* rot, int64_t rot_rows,
                          int64_t half, const int64_t* positions, const float* q_norm, const float* k_norm,
                          void* cache, int64_t batch, int64_t seq, int64_t max_len, int64_t heads, int64_t kv_heads,
                          int64_t dk, int64_t vp, int64_t dim, float eps, int dtype, void* stream) {
    MIX_TRY(check_dtype("gqa_append", dtype));
    MIX_TRY(check_ptrs("gqa_append", (const void*)proj, (const void*)cache));
    if (!positions) return fail(ASTRAI_MIX_BAD_ARG, "gqa_append: null pointer");
    MIX_TRY(check_gqa("gqa_append", heads, kv_heads, dk, vp));
    MIX_TRY(check_block("gqa_append", batch, seq, max_len, ld, heads * dk));
    if (rot) MIX_TRY(check_ptrs("gqa_append", (const void*)rot));
    if ((q_norm == nullptr) != (k_norm == nullptr)) return fail(ASTRAI_MIX_BAD_ARG, "gqa_append: one norm weight");
    if (q_norm) MIX_TRY(check_ptrs("gqa_append", (const void*)q_norm, (const void*)k_norm));
    if (k_off < heads * dk || v_off < heads * dk || k_off % 8 || v_off % 8 || k_off + kv_heads * dk > ld ||
        v_off + kv_heads * vp > ld || dim <= 0 || dim > dk || (rot && (half <= 0 || 2 * half > dim || rot_rows <= 0)) ||
        batch * seq * (heads + 2 * kv_heads) > kMaxInt)
        return fail(ASTRAI_MIX_BAD_ARG, "gqa_append: bad columns (k %lld, v %lld, half %lld, dim %lld)", (long long)k_off,
                    (long long)v_off, (long long)half, (long long)dim);
    if (dk > 512 || vp > 512) return fail(ASTRAI_MIX_UNSUPPORTED, "gqa_append: head sizes %lld, %lld (at most 512)",
                                          (long long)dk, (long long)vp);
    const GqaAppendArgs a = {proj, ld, (int)k_off, (int)v_off, rot, positions, q_norm, k_norm, cache, batch * seq, rot_rows,
                             (int)seq, (int)max_len, (int)half, (int)dim, eps};
    launch_gqa_append(a, gqa_dims(heads, kv_heads, dk, vp, 1, 1.0f, 0.0f, 0), dtype, static_cast<hipStream_t>(stream));
    return check_launch("gqa_append");
}

int astrai_mix_gqa_prefill(const void* proj, int64_t ld, int64_t g_off, const void* cache, void* out, int64_t batch,
                           int64_t seq, int64_t max_len, int64_t start, int64_t heads, int64_t kv_heads, int64_t dk,
                           int64_t vp, int64_t window, float scale, float softcap, int sink, void* stream) {
    MIX_TRY(check_ptrs("gqa_prefill", proj, cache, (const void*)out));
    MIX_TRY(check_gqa("gqa_prefill", heads, kv_heads, dk, vp));
    MIX_TRY(check_block("gqa_prefill", batch, seq, max_len, ld, heads * dk));
    MIX_TRY(check_gate("gqa_prefill", ld, g_off, heads * vp));
    if (window <= 0 || start < 0 || start + seq > max_len)
        return fail(ASTRAI_MIX_BAD_ARG, "gqa_prefill: tokens %lld .. %lld of %lld, window %lld", (long long)start,
                    (long long)(start + seq - 1), (long long)max_len, (long long)window);
    const LatentDims d = dims(heads, dk, 0, 32, vp, window, scale);
    if (!gqa_prefill_supported(d) || ((seq + 127) / 128) * batch * heads > kMaxInt)
        return fail(ASTRAI_MIX_UNSUPPORTED, "gqa_prefill: head sizes %lld, %lld (at most 128) or scale %g", (long long)dk,
                    (long long)vp, (double)scale);
    LatentPrefillArgs a;
    a.proj = proj;
    a.ld = ld;
    a.g_off = g_off < 0 ? -1 : (int)g_off;
    a.kv = a.cache = cache;
    a.out = out;
    a.batch = (int)batch;
    a.seq = (int)seq;
    a.max_len = a.n_keys = (int)max_len;
    a.start = (int)start;
    a.key_base = 0;
    a.group = (int)(heads / kv_heads);
    a.softcap = softcap;
    a.sink = sink;
    launch_gqa_prefill(a, d, static_cast<hipStream_t>(stream));
    return check_launch("gqa_prefill");
}

int64_t astrai_mix_gqa_rows_workspace_floats(int64_t tokens, int64_t heads, int64_t vp, int64_t nsplit) {
    return gqa_rows_workspace_floats(gqa_dims(heads, heads, 32, vp, 1, 1.0f, 0.0f, 0), tokens, (int)nsplit);
}

int astrai_mix_gqa_rows(const void* proj, int64_t ld, int64_t g_off, const void* cache, const int64_t* positions,
                        float* ws, void* out, int64_t batch, int64_t seq, int64_t max_len, int64_t heads,
                        int64_t kv_heads, int64_t dk, int64_t vp, int64_t window, float scale, float softcap, int sink,
                        int64_t nsplit, void* stream) {
    MIX_TRY(check_ptrs("gqa_rows", proj, cache, (const void*)ws, (const void*)out));
    if (!positions) return fail(ASTRAI_MIX_BAD_ARG, "gqa_rows: null pointer");
    MIX_TRY(check_gqa("gqa_rows", heads, kv_heads, dk, vp));
    MIX_TRY(check_block("gqa_rows", batch, seq, max_len, ld, heads * dk));
    MIX_TRY(check_gate("gqa_rows", ld, g_off, heads * vp));
    if (window <= 0 || nsplit < 1 || nsplit > kMaxSplit)
        return fail(ASTRAI_MIX_BAD_ARG, "gqa_rows: bad window or nsplit %lld", (long long)nsplit);
    const GqaDims d = gqa_dims(heads, kv_heads, dk, vp, window, scale, softcap, sink);
    if (!gqa_rows_mfma_supported(d) || seq * (heads / kv_heads) * nsplit > kMaxInt ||
        (max_len + 64) * kv_heads * (dk + vp) * 2 >= kMaxInt)
        return fail(ASTRAI_MIX_UNSUPPORTED, "gqa_rows: head sizes %lld, %lld (at most 256, 128), too many rows or a sequence of "
                    "2 GiB", (long long)dk, (long long)vp);
    const GqaRowsArgs a = {proj, ld, g_off < 0 ? -1 : (int)g_off, cache, positions, ws, out, (int)batch, (int)seq,
                           (int)max_len, (int)nsplit};
    launch_gqa_rows_mfma(a, d, static_cast<hipStream_t>(stream));
    return check_launch("gqa_rows");
}

int astrai_mix_gqa_rows_general(const void* proj, int64_t ld, int64_t g_off, const void* cache,
                                const int64_t* positions, void* out, int64_t batch, int64_t seq, int64_t max_len,
                                int64_t heads, int64_t kv_heads, int64_t dk, int64_t vp, int64_t window, float scale,
                                float softcap, int sink, int dtype, void* stream) {
    MIX_TRY(check_dtype("gqa_rows_general", dtype));
    MIX_TRY(check_ptrs("gqa_rows_general", proj, cache, (const void*)out));
    if (!positions) return fail(ASTRAI_MIX_BAD_ARG, "gqa_rows_general: null pointer");
    MIX_TRY(check_gqa("gqa_rows_general", heads, kv_heads, dk, vp));
    MIX_TRY(check_block("gqa_rows_general", batch, seq, max_len, ld, heads * dk));
    MIX_TRY(check_gate("gqa_rows_general", ld, g_off, heads * vp));
    if (window <= 0) return fail(ASTRAI_MIX_BAD_ARG, "gqa_rows_general: bad window");
    const GqaDims d = gqa_dims(heads, kv_heads, dk, vp, window, scale, softcap, sink);
    if (!gqa_rows_general_supported(d))
        return fail(ASTRAI_MIX_UNSUPPORTED, "gqa_rows_general: head sizes %lld, %lld (at most 1024)", (long long)dk, (long long)vp);
    const GqaRowsArgs a = {proj, ld, g_off < 0 ? -1 : (int)g_off, cache, positions, nullptr, out, (int)batch, (int)seq,
                           (int)max_len, 1};
    launch_gqa_rows_general(a, d, dtype, static_cast<hipStream_t>(stream));
    return check_launch("gqa_rows_general");
}

int astrai_mix_conv(const void* proj, int64_t ld, int64_t off, int64_t cols, const float* w, const float* bias,
                    int64_t taps, void* ring, const int64_t* positions, void* out, int64_t batch, int64_t seq, int silu,
                    int tail, int dtype, void* stream) {
    MIX_TRY(check_dtype("conv", dtype));
    MIX_TRY(check_ptrs("conv", proj));
    if (out) MIX_TRY(check_ptrs("conv", (const void*)out));
    MIX_TRY(check_block("conv", batch, seq, seq, ld, 8));
    MIX_TRY(check_conv("conv", ld, off, cols, w, bias, taps, ring, positions));
    if (batch * seq * (cols / 4) > (int64_t)kMaxInt * 64) return fail(ASTRAI_MIX_BAD_ARG, "conv: too many elements");
    const ConvArgs a = conv_args(proj, ld, off, cols, w, bias, taps, ring, positions, out, batch, seq, silu);
    if (out) launch_conv(a, dtype, static_cast<hipStream_t>(stream));
    if (tail) launch_conv_tail(a, dtype, static_cast<hipStream_t>(stream));
    return check_launch("conv");
}

int astrai_mix_rglru_chunk(const void* u, const void* proj, int64_t ld, int64_t y_off, const void* w_r, const void* w_i,
                           const float* b_r, const float* b_i, const float* coef, float* state, float* scratch,
                           void* out, int64_t batch, int64_t seq, int64_t blocks, int64_t bp, int64_t nseg,
                           void* stream) {
    MIX_TRY(check_ptrs("rglru_chunk", u, proj, w_r, w_i, (const void*)b_r, (const void*)b_i, (const void*)coef,
                       (const void*)state, (const void*)out));
    MIX_TRY(check_rglru("rglru_chunk", ld, y_off, batch, seq, blocks, bp));
    if (nseg < 1 || nseg > seq || (nseg > 1 && !scratch) || blocks * ((bp + 63) / 64) > kMaxGridYZ)
        return fail(ASTRAI_MIX_BAD_ARG, "rglru_chunk: bad nseg %lld or too many blocks", (long long)nseg);
    if (!rglru_chunk_supported((int)bp))
        return fail(ASTRAI_MIX_UNSUPPORTED, "rglru_chunk: blocks of %lld (at most 1024)", (long long)bp);
    launch_rglru_chunk(rglru_args(u, proj, ld, y_off, w_r, w_i, b_r, b_i, coef, state, scratch, out, batch, seq, blocks,
                                  bp, nseg), static_cast<hipStream_t>(stream));
    return check_launch("rglru_chunk");
}

int astrai_mix_rglru_general(const void* u, const void* proj, int64_t ld, int64_t y_off, const void* w_r,
                             const void* w_i, const float* b_r, const float* b_i, const float* coef, float* state,
                             float* scratch, void* out, int64_t batch, int64_t seq, int64_t blocks, int64_t bp,
                             int dtype, void* stream) {
    MIX_TRY(check_dtype("rglru_general", dtype));
    MIX_TRY(check_ptrs("rglru_general", u, proj, w_r, w_i, (const void*)b_r, (const void*)b_i, (const void*)coef,
                       (const void*)state, (const void*)scratch, (const void*)out));
    MIX_TRY(check_rglru("rglru_general", ld, y_off, batch, seq, blocks, bp));
    if (batch * seq * blocks * bp > (int64_t)kMaxInt * 256) return fail(ASTRAI_MIX_BAD_ARG, "rglru_general: too many elements");
    launch_rglru_general(rglru_args(u, proj, ld, y_off, w_r, w_i, b_r, b_i, coef, state, scratch, out, batch, seq,
                                    blocks, bp, 1), dtype, static_cast<hipStream_t>(stream));
    return check_launch("rglru_general");
}

int astrai_mix_rglru_step(const void* proj, int64_t ld, int64_t y_off, int64_t x_off, const float* conv_w,
                          const float* conv_b, int64_t taps, void* ring, const int64_t* positions, const void* w_r,
                          const void* w_i, const float* b_r, const float* b_i, const float* coef, float* state,
                          void* out, int64_t batch, int64_t seq, int64_t blocks, int64_t bp, void* stream) {
    MIX_TRY(check_ptrs("rglru_step", proj, w_r, w_i, (const void*)b_r, (const void*)b_i, (const void*)coef,
                       (const void*)state, (const void*)out));
    MIX_TRY(check_rglru("rglru_step", ld, y_off, batch, seq, blocks, bp));
    MIX_TRY(check_conv("rglru_step", ld, x_off, blocks * bp, conv_w, conv_b, taps, ring, positions));
    if (!rglru_step_supported((int)bp, (int)seq))
        return fail(ASTRAI_MIX_UNSUPPORTED, "rglru_step: %lld tokens (at most %d)", (long long)seq, kRingSteps);
    RglruArgs a = rglru_args(nullptr, proj, ld, y_off, w_r, w_i, b_r, b_i, coef, state, nullptr, out, batch, seq,
                             blocks, bp, 1);
    a.conv = conv_args(proj, ld, x_off, blocks * bp, conv_w, conv_b, taps, ring, positions, nullptr, batch, seq, 0);
    launch_rglru_step(a, static_cast<hipStream_t>(stream));
    return check_launch("rglru_step");
}

int astrai_mix_delta_step(const void* qkv, const void* proj, int64_t ld, int64_t x_off, int64_t b_off,
                          const float* conv_w, int64_t taps, void* ring, const int64_t* positions, const float* z,
                          const float* dt_bias, const float* decay, const void* gate, int64_t ldg, const float* norm_w,
                          float* state, void* out, int64_t batch, int64_t seq, int64_t heads, int64_t kv_heads,
                          int64_t dp, int64_t vp, int64_t vdim, float q_scale, float eps, int dtype, void* stream) {
    MIX_TRY(check_dtype("delta_step", dtype));
    MIX_TRY(check_ptrs("delta_step", proj, (const void*)z, (const void*)dt_bias, (const void*)decay, gate,
                       (const void*)norm_w, (const void*)state, (const void*)out));
    MIX_TRY(check_delta("delta_step", ld, b_off, batch, seq, heads, kv_heads, dp, vp));
    const int64_t cols = 2 * kv_heads * dp + heads * vp;
    if (qkv) MIX_TRY(check_ptrs("delta_step", qkv));
    else MIX_TRY(check_conv("delta_step", ld, x_off, cols, conv_w, nullptr, taps, ring, positions));
    if (ldg % 4 || ldg < heads * vp || vdim <= 0 || vdim > vp)
        return fail(ASTRAI_MIX_BAD_ARG, "delta_step: bad gate stride %lld or value size %lld", (long long)ldg, (long long)vdim);
    if (!delta_step_supported((int)dp, (int)vp) || (!qkv && seq > kRingSteps))
        return fail(ASTRAI_MIX_UNSUPPORTED, "delta_step: head sizes %lld, %lld or %lld tokens", (long long)dp, (long long)vp,
                    (long long)seq);
    DeltaArgs a = {};
    a.qkv = qkv;
    a.ldq = cols;
    a.proj = proj;
    a.ld = ld;
    a.b_off = (int)b_off;
    a.z = z;
    a.dt_bias = dt_bias;
    a.decay = decay;
    a.gate = gate;
    a.ldg = ldg;
    a.norm_w = norm_w;
    a.state = state;
    a.out = out;
    a.batch = (int)batch;
    a.seq = (int)seq;
    a.heads = (int)heads;
    a.kv_heads = (int)kv_heads;
    a.dp = (int)dp;
    a.vp = (int)vp;
    a.vdim = (int)vdim;
    a.q_scale = q_scale;
    a.eps = eps;
    if (!qkv) a.conv = conv_args(proj, ld, x_off, cols, conv_w, nullptr, taps, ring, positions, nullptr, batch, seq, 1);
    launch_delta_step(a, !qkv, dtype, static_cast<hipStream_t>(stream));
    return check_launch("delta_step");
}

int64_t astrai_mix_delta_image_bytes(int64_t dp) { return dp > 0 && dp <= 256 ? delta_image_bytes((int)dp) : 0; }

int astrai_mix_delta_chunk(const void* qkv, const void* proj, int64_t ld, int64_t b_off, const float* z,
                           const float* dt_bias, const float* decay, float* state, void* image, void* out, int64_t batch,
                           int64_t seq, int64_t heads, int64_t kv_heads, int64_t dp, int64_t vp, float q_scale,
                           void* stream) {
    MIX_TRY(check_ptrs("delta_chunk", qkv, proj, (const void*)z, (const void*)dt_bias, (const void*)decay,
                       (const void*)state, (const void*)image, (const void*)out));
    MIX_TRY(check_delta("delta_chunk", ld, b_off, batch, seq, heads, kv_heads, dp, vp));
    if (batch > kMaxGridYZ) return fail(ASTRAI_MIX_BAD_ARG, "delta_chunk: batch %lld", (long long)batch);
    if (!delta_chunk_supported((int)dp, (int)vp))
        return fail(ASTRAI_MIX_UNSUPPORTED, "delta_chunk: head size %lld (at most 256)", (long long)dp);
    DeltaArgs a = {};
    a.qkv = qkv;
    a.ldq = 2 * kv_heads * dp + heads * vp;
    a.proj = proj;
    a.ld = ld;
    a.b_off = (int)b_off;
    a.z = z;
    a.dt_bias = dt_bias;
    a.decay = decay;
    a.state = state;
    a.image = image;
    a.out = out;
    a.batch = (int)batch;
    a.seq = (int)seq;
    a.heads = (int)heads;
    a.kv_heads = (int)kv_heads;
    a.dp = (int)dp;
    a.vp = (int)vp;
    a.q_scale = q_scale;
    launch_delta_chunk(a, static_cast<hipStream_t>(stream));
    return check_launch("delta_chunk");
}

}  // extern "C"
