/* C ABI of libastrai_mix.so: sequence mixers (latent attention, lightning attention, grouped-query
 * attention with a sink, the real-gated linear recurrent unit, the gated delta rule) and the row
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

#define ASTRAI_MIX_ABI_VERSION 2

#define ASTRAI_MIX_OK 0
#define ASTRAI_MIX_BAD_ARG 1
#define ASTRAI_MIX_UNSUPPORTED 2
#define ASTRAI_MIX_LAUNCH_FAILED 3

#define ASTRAI_MIX_BF16 0
#define ASTRAI_MIX_F32 1

#define ASTRAI_MIX_LIGHTNING_CHUNK 64
#define ASTRAI_MIX_MAX_SPLIT 64
#define ASTRAI_MIX_RING_STEPS 8
#define ASTRAI_MIX_DELTA_CHUNK 16

#define ASTRAI_MIX_SILU 0
#define ASTRAI_MIX_GELU 1 /* tanh form */

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

/* x_out = mult * (y, or with tokens the rows y[tokens]) + x_in + u + vec, every term but the first optional
 * (null); h = x_out / sqrt(mean(x_out^2) + eps) * w, or x_out itself without w. y [rows or vocab, ldy] and u
 * [rows, ldu] are dtype, or float with y_float; vec, w float [width]; h dtype [rows, width]. */
int astrai_mix_sum_norm(const void* y, int64_t ldy, const int64_t* tokens, int64_t vocab, float mult, const float* x_in,
                        const void* u, int64_t ldu, const float* vec, float* x_out, const float* w, void* h,
                        int64_t rows, int64_t width, float eps, int y_float, int dtype, void* stream);

/* h = act(gate) * up; gu [rows, 2 ff] (gate columns, then up), ff % 8 == 0. */
int astrai_mix_act_mul(const void* gu, void* h, int64_t rows, int64_t ff, int act, int dtype, void* stream);

/* out = o / sqrt(mean(o^2) + eps) * w * sigmoid(g); the mean over `count` of the n columns (the
 * others are padding). g rows have stride ldg. n % 4 == 0, ldg % 4 == 0. */
int astrai_mix_gated_rms_norm(const void* o, const void* g, int64_t ldg, const float* w, void* out,
                              int64_t rows, int64_t n, int64_t count, float eps, int dtype, void* stream);

/* The same for each of `heads` groups of vp columns, w [vp], the mean over `count` of a group's columns. */
int astrai_mix_head_gated_rms_norm(const void* o, const void* g, int64_t ldg, const float* w, void* out, int64_t rows,
                                   int64_t heads, int64_t vp, int64_t count, float eps, int dtype, void* stream);

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

/* Grouped-query attention, after the input projection. proj [batch * seq, ld]: heads x dk query columns at 0,
 * kv_heads x dk key columns at k_off, kv_heads x vp value columns at v_off; dk, vp padded to multiples of 32.
 * A cached row is kv_heads x [key dk | value vp]. Query head h reads key/value head h / (heads / kv_heads).
 * _append: RMS norm of queries (in place) and keys over `dim` columns with weights q_norm, k_norm [dk] (both null:
 * none), rotation of pairs i, i + half (rot null: none), keys and values into cache [batch, max_len, ...] at
 * positions [seq]. */
int astrai_mix_gqa_append(void* proj, int64_t ld, int64_t k_off, int64_t v_off, const float* rot, int64_t rot_rows,
                          int64_t half, const int64_t* positions, const float* q_norm, const float* k_norm,
                          void* cache, int64_t batch, int64_t seq, int64_t max_len, int64_t heads, int64_t kv_heads,
                          int64_t dk, int64_t vp, int64_t dim, float eps, int dtype, void* stream);

/* out [batch * seq, heads * vp] of the new tokens' queries. Scores q . k * scale, softcap * tanh(score / softcap) if
 * softcap > 0; query p sees keys p - window + 1 .. p; with sink the softmax denominator has one more term exp(0);
 * with g_off >= 0 the output is multiplied by sigmoid of the heads * vp columns of proj from there.
 * _prefill (bf16): a prompt at positions start ..; UNSUPPORTED unless dk, vp <= 128 and 1e-4 <= scale <= 1e4.
 * _rows (bf16): a few tokens, positions from the device, nsplit workgroups per context, ws scratch
 * (_workspace_floats); UNSUPPORTED unless dk <= 256, vp <= 128 and a sequence's cache stays below 2 GiB.
 * _rows_general: the same arithmetic on the vector ALU, bf16 or float, dk, vp <= 1024. */
int astrai_mix_gqa_prefill(const void* proj, int64_t ld, int64_t g_off, const void* cache, void* out, int64_t batch,
                           int64_t seq, int64_t max_len, int64_t start, int64_t heads, int64_t kv_heads, int64_t dk,
                           int64_t vp, int64_t window, float scale, float softcap, int sink, void* stream);
int64_t astrai_mix_gqa_rows_workspace_floats(int64_t tokens, int64_t heads, int64_t vp, int64_t nsplit);
int astrai_mix_gqa_rows(const void* proj, int64_t ld, int64_t g_off, const void* cache, const int64_t* positions,
                        float* ws, void* out, int64_t batch, int64_t seq, int64_t max_len, int64_t heads,
                        int64_t kv_heads, int64_t dk, int64_t vp, int64_t window, float scale, float softcap, int sink,
                        int64_t nsplit, void* stream);
int astrai_mix_gqa_rows_general(const void* proj, int64_t ld, int64_t g_off, const void* cache,
                                const int64_t* positions, void* out, int64_t batch, int64_t seq, int64_t max_len,
                                int64_t heads, int64_t kv_heads, int64_t dk, int64_t vp, int64_t window, float scale,
                                float softcap, int sink, int dtype, void* stream);

/* Causal convolution per channel of the `cols` columns of proj [batch * seq, ld] from `off`:
 * out [batch * seq, cols] = act(bias + sum_j w[j] x(t - taps + 1 + j)), w float [taps, cols], bias float [cols] or
 * null, act silu or (silu = 0) none. ring [batch, taps - 1 + RING_STEPS, cols] holds earlier inputs, the one of position
 * p in row p modulo the rows; inputs before position 0 are zeros. out null: no output. tail: the block's last
 * taps - 1 inputs go into the ring (after the convolution, in stream order). cols % 4 == 0. */
int astrai_mix_conv(const void* proj, int64_t ld, int64_t off, int64_t cols, const float* w, const float* bias,
                    int64_t taps, void* ring, const int64_t* positions, void* out, int64_t batch, int64_t seq, int silu,
                    int tail, int dtype, void* stream);

/* Real-gated linear recurrent unit on u, blocks x bp channels (bp a multiple of 32):
 *   r, i = sigmoid(W u + b) per block, a = exp(coef r), S <- a S + sqrt(1 - a^2) i u, out = S gelu(y),
 * y columns of proj from y_off, b_r, b_i, coef (<= 0), state [batch, channels] float.
 * _chunk (bf16, bp <= 1024): w [blocks, out, in]; nseg segments of the sequence side by side, scratch
 * [batch, nseg, 2, channels] float when nseg > 1; a segment is a whole number of tiles of 64 tokens.
 * _general (bf16 or float): w [blocks, in, out], scratch [2, batch * seq, channels].
 * _step (bf16, seq <= RING_STEPS): convolves proj's columns from x_off itself and updates the ring (as above). */
int astrai_mix_rglru_chunk(const void* u, const void* proj, int64_t ld, int64_t y_off, const void* w_r, const void* w_i,
                           const float* b_r, const float* b_i, const float* coef, float* state, float* scratch,
                           void* out, int64_t batch, int64_t seq, int64_t blocks, int64_t bp, int64_t nseg,
                           void* stream);
int astrai_mix_rglru_general(const void* u, const void* proj, int64_t ld, int64_t y_off, const void* w_r,
                             const void* w_i, const float* b_r, const float* b_i, const float* coef, float* state,
                             float* scratch, void* out, int64_t batch, int64_t seq, int64_t blocks, int64_t bp,
                             int dtype, void* stream);
int astrai_mix_rglru_step(const void* proj, int64_t ld, int64_t y_off, int64_t x_off, const float* conv_w,
                          const float* conv_b, int64_t taps, void* ring, const int64_t* positions, const void* w_r,
                          const void* w_i, const float* b_r, const float* b_i, const float* coef, float* state,
                          void* out, int64_t batch, int64_t seq, int64_t blocks, int64_t bp, void* stream);

/* Gated delta rule with one decay per key channel, state [batch, heads, dp, vp] float:
 *   S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q,
 * k a unit vector, q a unit vector times q_scale (both x / sqrt(sum x^2 + 1e-6)), head h using q/k head
 * h / (heads / kv_heads); beta the sigmoid of proj's column b_off + h; g = exp(-decay_h softplus(z + dt_bias)), z float
 * [batch * seq, heads * dp]. qkv [batch * seq, 2 kv_heads dp + heads vp]: q | k | v after convolution and silu.
 * _step (bf16 or float): out = o / sqrt(mean(o^2) + eps) * norm_w * sigmoid(gate) per head (vdim real columns, gate rows
 * of stride ldg). qkv null (seq <= RING_STEPS): convolves proj's columns from x_off itself and updates the ring.
 * UNSUPPORTED unless vp <= 256 and dp * (vp / 4 rounded up to a power of two, at least 8) <= 16384.
 * _chunk (bf16, dp <= 256): out = o; image: delta_image_bytes * batch * heads * ceil(seq / DELTA_CHUNK) bytes. */
int astrai_mix_delta_step(const void* qkv, const void* proj, int64_t ld, int64_t x_off, int64_t b_off,
                          const float* conv_w, int64_t taps, void* ring, const int64_t* positions, const float* z,
                          const float* dt_bias, const float* decay, const void* gate, int64_t ldg, const float* norm_w,
                          float* state, void* out, int64_t batch, int64_t seq, int64_t heads, int64_t kv_heads,
                          int64_t dp, int64_t vp, int64_t vdim, float q_scale, float eps, int dtype, void* stream);
int64_t astrai_mix_delta_image_bytes(int64_t dp);
int astrai_mix_delta_chunk(const void* qkv, const void* proj, int64_t ld, int64_t b_off, const float* z,
                           const float* dt_bias, const float* decay, float* state, void* image, void* out, int64_t batch,
                           int64_t seq, int64_t heads, int64_t kv_heads, int64_t dp, int64_t vp, float q_scale,
                           void* stream);

#ifdef __cplusplus
}
#endif

#endif /* ASTRAI_MIX_H */
