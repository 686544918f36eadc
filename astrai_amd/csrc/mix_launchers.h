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
void launch_silu_mul(const void* gu, void* h, int64_t rows, int ff, int dtype, hipStream_t stream);
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
};
// bf16 MFMA kernel; false if the head sizes are not covered
bool latent_prefill_supported(const LatentDims& d);
bool launch_latent_prefill(const LatentPrefillArgs& a, const LatentDims& d, hipStream_t stream);

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

}  // namespace astrai_mix
