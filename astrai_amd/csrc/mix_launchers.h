// Internal interface between mix_abi.hip and the kernels of libastrai_mix.so. dtype: 0 = bf16,
// 1 = float (activations, weights and cached latents); norm weights, the residual stream, rotary
// tables and recurrent states are float in both.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

namespace astrai_mix {

// ---- mix_rows.hip ---------------------------------------------------------------------------
struct ResidualNormArgs {
    const void* y;          // [rows, width], or the embedding table [vocab, width] with `tokens`
    const int64_t* tokens;  // [rows] or null
    const float* x_in;      // [rows, width] (unused with tokens)
    float* x_out;           // [rows, width], may be x_in
    const float* w_post;    // [width] (unused with tokens)
    const float* w_pre;     // [width]
    void* h;                // [rows, width]
    int64_t rows, vocab;
    int width;
    float mult, eps;
};
void launch_residual_norm(const ResidualNormArgs& a, int dtype, hipStream_t stream);

struct SumNormArgs {
    const void* y;          // [rows, ldy], or the embedding table [vocab, ldy] with `tokens`
    int64_t ldy;
    const int64_t* tokens;  // [rows] or null
    const float* x_in;      // [rows, width] or null
    const void* u;          // [rows, ldu] or null, of y's type
    int64_t ldu;
    const float* vec;       // [width] or null
    float* x_out;           // [rows, width], may be x_in
    const float* w;         // [width], or null: no norm
    void* h;                // [rows, width]
    int64_t rows, vocab;
    int width;
    float mult, eps;        // mult multiplies y
};
// y_float: y and u are float with bf16 h
void launch_sum_norm(const SumNormArgs& a, int dtype, bool y_float, hipStream_t stream);

constexpr int kActSilu = 0, kActGelu = 1;   // gelu in its tanh form
void launch_act_mul(const void* gu, void* h, int64_t rows, int ff, int act, int dtype, hipStream_t stream);

struct HeadNormArgs {
    const void* o;    // [rows, heads * vp]
    const void* g;    // [rows, ldg]
    int64_t ldg;
    const float* w;   // [vp]
    void* out;        // [rows, heads * vp]
    int64_t rows;
    int heads, vp, count;
    float eps;
};
void launch_head_gated_rms_norm(const HeadNormArgs& a, int dtype, hipStream_t stream);
void launch_gated_rms_norm(const void* o, const void* g, int64_t ldg, const float* w, void* out, int64_t rows,
                           int n, int count, float eps, int dtype, hipStream_t stream);

// ---- mix_latent.hip / mix_latent_prefill.hip --------------------------------------------------
// Head sizes are padded: dn (unrotated), dr (rotated), rp (latent), vp (value) are multiples of 32
// whose padding is zero in the weights and therefore in every activation. A cached row is
// [latent rp | rotated key part dr].
struct LatentDims {
    int heads, dn, dr, rp, vp;
    int window;   // a query at position p sees keys p - window + 1 .. p
    float scale;
};

struct LatentAppendArgs {
    void* proj;                // [batch * seq, ld]: q (heads x (dn + dr)), then at dkv_off the latent rows
    int64_t ld;
    int dkv_off;               // < 0: no latent in this projection (the layer reads another layer's cache)
    const float* rot;          // [positions, half, 2] (cos, sin)
    const int64_t* positions;  // [seq]
    const float* norm_w;       // [rp]
    void* cache;               // [batch, max_len, rp + dr]
    const void* w_uk_t;        // [heads, rp, dn], with q_abs (bf16)
    void* q_abs;               // [batch * seq, heads, rp] or null
    int64_t tokens;            // batch * seq
    int64_t rot_rows;          // rows of `rot`
    int seq, max_len, half, kv_rank;
    float eps;
};
void launch_latent_append(const LatentAppendArgs& a, const LatentDims& d, int dtype, hipStream_t stream);

struct LatentPrefillArgs {
    const void* proj;    // as above, q rotated
    int64_t ld;
    int g_off;           // column of the per-head gate logits
    const void* kv;      // [batch, n_keys, heads * (dn + vp)]: per head unrotated key, value
    const void* cache;   // [batch, max_len, rp + dr]
    void* out;           // [batch, seq, heads * vp]
    int batch, seq, max_len;
    int start;           // position of the first new token
    int key_base;        // position of row 0 of kv
    int n_keys;
    // grouped-query heads: `group` query heads share a key / value head of kv, there is no rotated part
    int group = 1;
    float softcap = 0.0f;   // scores become softcap * tanh(score / softcap); 0: none
    int sink = 0;           // one more term exp(0) in the softmax denominator
};
// bf16 MFMA kernel; false if the head sizes are not covered
bool latent_prefill_supported(const LatentDims& d);
bool launch_latent_prefill(const LatentPrefillArgs& a, const LatentDims& d, hipStream_t stream);
// d.dr = 0; the gate is per element, heads * vp columns from g_off (< 0: no gate)
bool gqa_prefill_supported(const LatentDims& d);
bool launch_gqa_prefill(const LatentPrefillArgs& a, const LatentDims& d, hipStream_t stream);

constexpr int kMaxSplit = 64;
struct LatentRowsArgs {
    const void* proj;          // as above, q rotated
    int64_t ld;
    int g_off;
    const void* w_ukv;         // [heads * (dn + vp), rp]
    const void* cache;
    const int64_t* positions;  // [seq]
    const void* q_abs;         // [batch * seq, heads, rp] (MFMA path, as the next two)
    void* o_lat;               // scratch [batch * seq, heads, rp], may be q_abs
    float* ws;                 // scratch, latent_rows_workspace_floats
    void* out;                 // [batch, seq, heads * vp]
    int batch, seq, max_len, nsplit;
};
// attention in the latent space (queries absorbed through W_uk): MFMA kernels for bf16, else the
// general kernel
bool latent_rows_mfma_supported(const LatentDims& d);
int64_t latent_rows_workspace_floats(const LatentDims& d, int64_t tokens, int nsplit);
void launch_latent_rows_mfma(const LatentRowsArgs& a, const LatentDims& d, hipStream_t stream);
bool latent_rows_general_supported(const LatentDims& d);
void launch_latent_rows_general(const LatentRowsArgs& a, const LatentDims& d, int dtype, hipStream_t stream);

// ---- mix_lightning.hip ------------------------------------------------------------------------
constexpr int kLightningChunk = 64;
struct LightningArgs {
    const void* proj;     // [batch * seq, ld]: columns q (heads x dp), k (heads x dp), v (heads x vp)
    int64_t ld;
    int q_off, k_off, v_off;
    const float* decay_pow;  // [heads, kLightningChunk + 1]: decay^n
    float* state;         // [batch, heads, dp, vp], read and written
    float* seg_state;     // [batch, heads, nseg, dp, vp] scratch, nseg > 1
    void* out;            // [batch * seq, heads * vp]
    int batch, seq, heads, dp, vp;   // dp, vp padded to multiples of 32
    int nseg;             // segments of the sequence that run concurrently (chunk kernel)
};
// chunked form on the matrix cores, bf16; false if dp is not covered
bool lightning_chunk_supported(int dp, int vp);
bool launch_lightning_chunk(const LightningArgs& a, hipStream_t stream);
// token by token, state in registers
bool lightning_step_supported(int dp, int vp);
void launch_lightning_step(const LightningArgs& a, int dtype, hipStream_t stream);


// ---- mix_gqa.hip --------------------------------------------------------------------------------
// Grouped-query attention over cached keys and values. A cached row holds kv_heads x [key dk | value vp].
struct GqaDims {
    int heads, kv_heads, dk, vp;   // dk, vp padded to multiples of 32
    int window;                    // a query at position p sees keys p - window + 1 .. p
    float scale, softcap;          // softcap 0: none
    int sink;                      // one more term exp(0) in the softmax denominator
};

struct GqaAppendArgs {
    void* proj;                // [batch * seq, ld]: q (heads x dk) at 0, k (kv_heads x dk), v (kv_heads x vp)
    int64_t ld;
    int k_off, v_off;
    const float* rot;          // [positions, half, 2] (cos, sin), or null: no rotation
    const int64_t* positions;  // [seq]
    const float *q_norm, *k_norm;   // [dk], or null: no norm
    void* cache;               // [batch, max_len, kv_heads * (dk + vp)]
    int64_t tokens, rot_rows;
    int seq, max_len, half, dim;   // dim: the real columns of dk
    float eps;
};
void launch_gqa_append(const GqaAppendArgs& a, const GqaDims& d, int dtype, hipStream_t stream);

struct GqaRowsArgs {
    const void* proj;          // as above, q normed and rotated
    int64_t ld;
    int g_off;                 // heads x vp gate logits, < 0: no gate
    const void* cache;
    const int64_t* positions;
    float* ws;                 // gqa_rows_workspace_floats (MFMA path)
    void* out;                 // [batch, seq, heads * vp]
    int batch, seq, max_len, nsplit;
};
bool gqa_rows_mfma_supported(const GqaDims& d);
int64_t gqa_rows_workspace_floats(const GqaDims& d, int64_t tokens, int nsplit);
void launch_gqa_rows_mfma(const GqaRowsArgs& a, const GqaDims& d, hipStream_t stream);
bool gqa_rows_general_supported(const GqaDims& d);
void launch_gqa_rows_general(const GqaRowsArgs& a, const GqaDims& d, int dtype, hipStream_t stream);

// ---- mix_conv.hip ---------------------------------------------------------------------------------
// Causal convolution per channel. A ring holds the last inputs of every sequence, input of position p in
// row p % ring_rows; positions below 0 read as zeros.
constexpr int kRingSteps = 8;   // a ring has taps - 1 + kRingSteps rows: a step of that many tokens may read
                                // and write it at once
struct ConvArgs {
    const void* proj;          // [batch * seq, ld], `cols` columns from `off`
    int64_t ld;
    int off, cols;
    const float* taps_w;       // [taps, cols], last row: the current token's
    const float* bias;         // [cols] or null
    void* ring;                // [batch, ring_rows, cols]
    const int64_t* positions;  // [seq]
    void* out;                 // [batch * seq, cols]
    int batch, seq, taps, ring_rows;
    int silu;
};
void launch_conv(const ConvArgs& a, int dtype, hipStream_t stream);        // reads the ring
void launch_conv_tail(const ConvArgs& a, int dtype, hipStream_t stream);   // writes the last inputs into it

// ---- mix_rglru.hip --------------------------------------------------------------------------------
// S <- a S + sqrt(1 - a^2) i u per channel, a = exp(coef r), r and i sigmoids of block-diagonal products
// of u; out = S * gelu(y). Channels: blocks x bp, bp padded to a multiple of 32.
struct RglruArgs {
    const void* proj;     // [batch * seq, ld]
    int64_t ld;
    int y_off;
    const void* u;        // [batch * seq, blocks * bp], the convolved x (not for the fused step)
    const void *w_r, *w_i;       // [blocks, bp, bp], out by in
    const float *b_r, *b_i;      // [blocks * bp]
    const float* coef;           // [blocks * bp], -8 softplus(lam)
    float* state;                // [batch, blocks * bp], read and written
    float* scratch;              // general: [2, batch * seq, blocks * bp]; chunk with nseg > 1:
                                 // [batch, nseg, 2, blocks * bp]
    void* out;                   // [batch * seq, blocks * bp]
    int batch, seq, blocks, bp;
    int nseg;                    // segments of the sequence that run side by side (chunk)
    ConvArgs conv;               // fused step
};
bool rglru_chunk_supported(int bp);
void launch_rglru_chunk(const RglruArgs& a, hipStream_t stream);
bool rglru_step_supported(int bp, int seq);
void launch_rglru_step(const RglruArgs& a, hipStream_t stream);
// w_r, w_i transposed, [blocks, in, out]
void launch_rglru_general(const RglruArgs& a, int dtype, hipStream_t stream);

// ---- mix_delta.hip --------------------------------------------------------------------------------
// Gated delta rule with one decay per key channel. q, k: kv_heads x dp, v: heads x vp columns, consecutive.
constexpr int kDeltaChunk = 16;
struct DeltaArgs {
    const void* qkv;      // [batch * seq, ldq]: q | k | v after convolution and silu (from q_off)
    int64_t ldq;
    const void* proj;     // [batch * seq, ld]
    int64_t ld;
    int b_off;            // step-size logits, heads columns of proj
    const float* z;       // [batch * seq, heads * dp] decay logits
    const float* dt_bias;     // [heads * dp]
    const float* decay;       // [heads], exp(A_log)
    const void* gate;         // [batch * seq, ldg] output gate logits, heads x vp
    int64_t ldg;
    const float* norm_w;      // [vp]
    float* state;             // [batch, heads, dp, vp], read and written
    void* image;              // chunk: delta_image_bytes per (sequence, head, chunk)
    void* out;                // [batch * seq, heads * vp]
    int batch, seq, heads, kv_heads, dp, vp;   // dp, vp padded to multiples of 32
    float q_scale, eps;
    int vdim;                 // the real columns of vp
    ConvArgs conv;            // fused step
};
bool delta_step_supported(int dp, int vp);
// token by token, state in registers, normed and gated output; fused: convolves conv.proj itself
void launch_delta_step(const DeltaArgs& a, bool fused, int dtype, hipStream_t stream);
bool delta_chunk_supported(int dp, int vp);
int64_t delta_image_bytes(int dp);
// chunked form on the matrix cores, bf16; out is neither normed nor gated
void launch_delta_chunk(const DeltaArgs& a, hipStream_t stream);

}  // namespace astrai_mix
