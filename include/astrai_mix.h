/* C ABI of libastrai_mix.so: sequence mixers (latent attention, lightning attention) and the row
 * operations around them, for decoders with an fp32 residual stream, on gfx950.
 *
 * Every entry takes raw device pointers and a HIP stream, launches asynchronously, allocates
 * nothing and never synchronises (all of them may be captured into a HIP graph). Returns 0, or a
 * status with the reason in astrai_mix_last_error().
 *
 * dtype: 0 = bf16, 1 = float, the type of activations, matrix weights and cached latents (void*).
 * Norm weights, residual stream, rotary tables, decay powers and recurrent states are float.
 * Head sizes are given padded to multiples of 32; padding is zero in the weights, hence in every
 * activation. Pointers are 16-byte aligned.
 */
#ifndef ASTRAI_MIX_H
#define ASTRAI_MIX_H

#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define ASTRAI_MIX_ABI_VERSION 1

#define ASTRAI_MIX_OK 0
#define ASTRAI_MIX_BAD_ARG 1
#define ASTRAI_MIX_UNSUPPORTED 2
#define ASTRAI_MIX_LAUNCH_FAILED 3

#define ASTRAI_MIX_BF16 0
#define ASTRAI_MIX_F32 1

#define ASTRAI_MIX_LIGHTNING_CHUNK 64
#define ASTRAI_MIX_MAX_SPLIT 64

int astrai_mix_abi_version(void);
const char* astrai_mix_last_error(void);

/* x_out = x_in + mult * LN(y) * w_post; h = LN(x_out) * w_pre. y, h dtype [rows, width];
 * x_in, x_out float (may be the same); LN = layer norm with eps inside the root, no bias. */
int astrai_mix_residual_norm(const void* y, const float* x_in, float* x_out, const float* w_post,
                             const float* w_pre, void* h, int64_t rows, int64_t width, float mult,
                             float eps, int dtype, void* stream);

/* x_out = table[tokens]; h = LN(x_out) * w_pre. table dtype [vocab, width], tokens int64 [rows]
 * (ids outside the table are clamped into it). */
int astrai_mix_embed_norm(const void* table, const int64_t* tokens, float* x_out, const float* w_pre,
                          void* h, int64_t rows, int64_t width, int64_t vocab, float eps, int dtype,
                          void* stream);

/* h = silu(gate) * up; gu [rows, 2 ff] (gate columns, then up), ff % 8 == 0. */
int astrai_mix_silu_mul(const void* gu, void* h, int64_t rows, int64_t ff, int dtype, void* stream);

/* out = o / sqrt(mean(o^2) + eps) * w * sigmoid(g); the mean over `count` of the n columns (the
 * others are padding). g rows have stride ldg. n % 4 == 0, ldg % 4 == 0. */
int astrai_mix_gated_rms_norm(const void* o, const void* g, int64_t ldg, const float* w, void* out,
                              int64_t rows, int64_t n, int64_t count, float eps, int dtype, void* stream);

/* Latent attention, after the input projection. proj [batch * seq, ld]: heads x (dn + dr) query
 * columns, at dkv_off (>= 0) the rp + dr latent columns. Rotates the first 2 * half of every head's dr
 * rotated columns in place (pairs i, i + half; rot [rot_rows, half, 2] = cos, sin per position),
 * writes (RMS norm of the latent over kv_rank columns, rotated key part) into
 * cache [batch, max_len, rp + dr] at positions [seq]. dkv_off < 0: queries only. With q_abs (bf16
 * [batch * seq, heads, rp], else null): also q_abs = W_uk^T q_unrotated per head, w_uk_t
 * [heads, rp, dn] being W_uk's rows transposed. */
int astrai_mix_latent_append(void* proj, int64_t ld, int64_t dkv_off, const float* rot, int64_t rot_rows,
                             int64_t half, const int64_t* positions, const float* norm_w, void* cache,
                             const void* w_uk_t, void* q_abs, int64_t batch, int64_t seq, int64_t max_len,
                             int64_t heads, int64_t dn, int64_t dr, int64_t rp, int64_t kv_rank, float eps, int dtype, void* stream);

/* Sliding-window attention of seq new tokens at positions start .. start + seq - 1 (bf16). kv
 * [batch, n_keys, heads * (dn + vp)]: per head the unrotated key and the value of positions
 * key_base .. ; the rotated key part comes from the cache. Query p sees keys p - window + 1 .. p.
 * Head h's output is multiplied by sigmoid(proj[:, g_off + h]). out [batch, seq, heads * vp].
 * UNSUPPORTED unless dn <= 128, dr <= 64, vp <= 128 and 1e-4 <= scale <= 1e4. */
int astrai_mix_latent_prefill(const void* proj, int64_t ld, int64_t g_off, const void* kv, const void* cache,
                              void* out, int64_t batch, int64_t seq, int64_t max_len, int64_t start,
                              int64_t key_base, int64_t n_keys, int64_t heads, int64_t dn, int64_t dr,
                              int64_t rp, int64_t vp, int64_t window, float scale, void* stream);

/* The same for a few new tokens, attending in the latent space with the absorbed queries of
 * latent_append; W_uv is applied to the attended latent. w_ukv [heads * (dn + vp), rp]: per head the key
 * rows, then the value rows. Positions come from the device. nsplit workgroups share a context (1 ..
 * ASTRAI_MIX_MAX_SPLIT). bf16; q_abs is overwritten, ws (astrai_mix_latent_rows_workspace_floats)
 * scratch. UNSUPPORTED unless rp <= 1024, dr <= 64 and a sequence's cache stays below 2 GiB. */
int64_t astrai_mix_latent_rows_workspace_floats(int64_t tokens, int64_t heads, int64_t rp, int64_t nsplit);
int astrai_mix_latent_rows(const void* proj, int64_t ld, int64_t g_off, const void* w_ukv, const void* cache,
                           const int64_t* positions, void* q_abs, float* ws, void* out, int64_t batch,
                           int64_t seq, int64_t max_len, int64_t heads, int64_t dn, int64_t dr, int64_t rp,
                           int64_t vp, int64_t window, float scale, int64_t nsplit, void* stream);

/* The same arithmetic on the vector ALU, bf16 or float, rp <= 2048 and dr <= 512. */
int astrai_mix_latent_rows_general(const void* proj, int64_t ld, int64_t g_off, const void* w_ukv,
                                   const void* cache, const int64_t* positions, void* out, int64_t batch,
                                   int64_t seq, int64_t max_len, int64_t heads, int64_t dn, int64_t dr,
                                   int64_t rp, int64_t vp, int64_t window, float scale, int dtype, void* stream);

/* Lightning attention: S <- decay S + k v^T, o = S^T q per head, on silu of the projections.
 * proj [batch * seq, ld] with q (heads x dp) at q_off, k at k_off, v (heads x vp) at v_off;
 * decay_pow [heads, CHUNK + 1] = decay^0 .. decay^CHUNK; state [batch, heads, dp, vp] read and
 * written; out [batch * seq, heads * vp].
 * _chunk (bf16, dp <= 256): matrix-core form, nseg segments of the sequence side by side (at most
 * ceil(seq / CHUNK)), seg_state [batch, heads, nseg, dp, vp] scratch when nseg > 1.
 * _step (bf16 or float, dp <= 1024): token by token. */
int astrai_mix_lightning_chunk(const void* proj, int64_t ld, int64_t q_off, int64_t k_off, int64_t v_off,
                               const float* decay_pow, float* state, float* seg_state, void* out, int64_t batch,
                               int64_t seq, int64_t heads, int64_t dp, int64_t vp, int64_t nseg, void* stream);
int astrai_mix_lightning_step(const void* proj, int64_t ld, int64_t q_off, int64_t k_off, int64_t v_off,
                              const float* decay_pow, float* state, void* out, int64_t batch, int64_t seq,
                              int64_t heads, int64_t dp, int64_t vp, int dtype, void* stream);

#ifdef __cplusplus
}
#endif

#endif /* ASTRAI_MIX_H */
