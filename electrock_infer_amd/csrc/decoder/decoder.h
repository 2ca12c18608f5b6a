// Shared declarations of the decoder library: float32-stream row kernels, gated linear attention, recurrences with one decay
// per head, latent attention, softmax attention.
#pragma once
#include "../common.h"
#include "../../../include/electrock_decoder.h"

namespace em {

__device__ __forceinline__ float silu(float g) { return g / (1.0f + expf(-g)); }
__device__ __forceinline__ float gelu_tanh(float z) {
    return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// Lets a kernel take `bytes` of dynamic LDS (one CU has 160 KB); 0, or the runtime's error.
constexpr size_t kLdsPerCu = 160 * 1024;
inline int allow_lds(const void* kernel, size_t bytes) {
    if (bytes > kLdsPerCu) return EM_ERR_UNSUPPORTED;
    if (bytes <= 64 * 1024) return 0;
    return static_cast<int>(hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(bytes)));
}

// ---- rows.hip ----
bool row_width_ok(int W);
int launch_embed(const int32_t* tokens, const void* table, float scale, float* x, void* copy, int64_t copy_stride,
                 int64_t T, int W, int dtype, hipStream_t s);
int launch_residual_norm(int update, float* x, const void* y, int y_dtype, int y_parts, const float* post_w, const float* next_w,
                         void* out, int64_t out_stride, int64_t T, int W, float eps, int dtype, hipStream_t s);
int launch_relu_squared(void* u, int64_t n, int dtype, hipStream_t s);
int launch_silu_gate(const void* u, void* out, int64_t T, int ff, int dtype, hipStream_t s);
int launch_gated_norm(void* y, const void* z, int64_t z_stride, const float* w, int64_t T, int parts, int size, float eps, int dtype,
                      hipStream_t s);

// ---- skinny_gemm.hip ----
bool skinny_supported(int64_t T, int N, int K);
int skinny_splits(int T, int N, int K);
int launch_skinny_gemm(const void* x, const void* w, void* out, bool f32, int splits, int T, int N, int K, int act, hipStream_t s);

// ---- token_side.hip ----
struct TokenSideProblem {
    float* x;                // [T, W]
    const uint16_t* y;       // [T, W]
    const float *post_w, *side_norm, *next_w;
    const uint16_t *gate, *proj;   // [dim, W], [W, dim]
    const int32_t* tokens;
    const uint16_t* table;
    int64_t table_stride;
    int column0;
    uint16_t* out;
    int64_t out_stride;
    int64_t T;
    int W, dim;
    float eps;
    int rows_per_group, g_offset, part_offset;  // set by the launcher
};
int launch_token_gate(const void* x, const void* gate, const int32_t* tokens, const void* table, int64_t table_stride,
                      int column0, void* g, int64_t T, int W, int dim, int dtype, hipStream_t s);
bool token_side_supported(int W, int dim);
int launch_token_side(TokenSideProblem p, hipStream_t s);

// ---- gla.hip ----
struct GlaProblem {
    const void *q, *k, *v, *g, *a1;
    int64_t stride;
    const void* a2;
    int rank, a2_stride;
    const float* bias;
    float tau;
    const float* norm_w;
    void* out;
    float* bl;
    const int32_t* chunks;
    const int32_t *slots, *starts;
    float *states, *chunk_states, *chunk_decay;
    int heads, dim, vdim;
    float q_scale, eps;
    int dtype;
};
bool gla_supported(int heads, int dim, int vdim, int rank);
int launch_gla_prefill(const GlaProblem& g, const int32_t* seq_chunks, int n_chunks, int n_seqs, int chunk_tokens,
                       hipStream_t s);
int launch_gla_step(const GlaProblem& g, int n_seqs, hipStream_t s);

// ---- recurrence.hip ----
struct RecurProblem {
    const void *q, *k, *v;       // projections: q, k head g at g * dim, v head h at h * vdim
    const void *decay_in, *beta_in, *gate;   // column h, column h (null: additive rule), head h at h * vdim (delta rule)
    int64_t stride;              // of all of these
    const float *conv_w, *conv_b;            // [channels, taps], [channels] or null; channels: q, k, v
    const float *a_log, *dt_bias, *skip, *norm_w;   // [heads], [heads], [heads] or null, [vdim] (delta rule)
    void* ring;                  // [slots, taps, channels]
    float* states;               // [slots, heads, dim, vdim]
    void* out;                   // [T, heads * vdim]
    const int32_t *slots, *starts, *q_begin;
    const int4* chunks;
    const int32_t* seq_chunks;
    float *q_f, *k_f;            // [T, kv_heads, dim padded to 16]
    void* v_f;                   // [T, heads * vdim]
    float *rates, *blocks, *chunk_states, *chunk_trans;
    int n_seqs, n_chunks, chunk_tokens;
    int heads, kv_heads, dim, vdim, taps, dtype;
    float q_scale, unit_eps, eps;
};
bool recur_supported(int heads, int kv_heads, int dim, int vdim, int taps);
__host__ __device__ constexpr int recur_record(bool delta) { return delta ? 576 : 320; }   // floats of a block's record
int launch_recur_prefill(const RecurProblem& p, hipStream_t s);
int launch_recur_step(const RecurProblem& p, hipStream_t s);

// ---- attention.hip ----
struct AttnProblem {
    const void *q, *k, *v;       // projections, heads next to each other
    int64_t stride;
    const void* v_first;         // rows of the values that are mixed in
    int64_t v_first_stride;
    const float* mix;            // their share, a number in device memory; null: none
    const float *q_norm, *k_norm;   // [dim] or null
    const float* inv_freq;       // [rot / 2]
    const int32_t *positions, *cache_rows;
    void* cache;                 // [rows, attn_row_elems]
    void* q_out;                 // [T, heads, attn_pitch(dim)]
    void* out;                   // [T, heads * vdim]
    const int32_t *q_begin, *starts, *tables;
    int table_width, block_size;
    int heads, kv_heads, dim, vdim, rot, window, dtype;
    float scale, softcap, eps;
};
__host__ __device__ constexpr int attn_pitch(int dim) { return (dim + 7) / 8 * 8; }
__host__ __device__ constexpr int attn_row_elems(int kv_heads, int dim, int vdim) { return kv_heads * (attn_pitch(dim) + attn_pitch(vdim)); }
constexpr int kAttnMaxSplits = 64;
bool attn_supported(int heads, int kv_heads, int dim, int vdim, int rot);
bool attn_prompt_supported(int dim, int vdim);
int launch_attn_prepare(const AttnProblem& p, int64_t T, hipStream_t s);
int launch_attn_paged(const AttnProblem& p, int n_seqs, int max_q, int splits, float* part_o, float* part_ml, int64_t T, hipStream_t s);
int launch_attn_prompt(const AttnProblem& p, int n_seqs, int max_q, hipStream_t s);

// ---- latent_attention.hip ----
struct LatentProblem {
    void* q;                 // projection rows: head h at h * (dim + rot), rotated in place by the prepare step
    int64_t q_stride;
    const void* down;        // latent + rotated key part of every token, before norm and rotation
    int64_t down_stride;
    const float* latent_w;   // [rank]
    const float* inv_freq;   // [rot / 2]
    const int32_t* positions;
    const int32_t* cache_rows;   // row of the cache that takes every token
    void* cache;             // [rows, latent_row_elems]
    const void* q_latent;    // [T, heads, latent_pitch]
    void* out;               // [T, heads, latent_pitch]
    const float* sink;       // [heads]
    const int32_t *q_begin, *starts, *tables;
    int table_width, block_size;
    int heads, dim, rot, rank;
    float scale, eps;
    int dtype;
};
__host__ __device__ constexpr int latent_pitch(int rank) { return (rank + 7) / 8 * 8; }
__host__ __device__ constexpr int latent_row_elems(int rank, int rot) { return latent_pitch(rank) + (rot + 7) / 8 * 8; }
constexpr int kLatentMaxSplits = 256;
bool latent_supported(int heads, int dim, int rot, int rank);
int launch_latent_prepare(const LatentProblem& p, int64_t T, hipStream_t s);
int launch_latent_paged(const LatentProblem& p, int n_seqs, int max_q, int splits, float* part_o, float* part_ml,
                        int64_t T, hipStream_t s);
int launch_head_gemm(const void* a, int64_t a_row, int64_t a_head, const void* b, void* out, int64_t o_row,
                     int64_t o_head, int64_t T, int heads, int N, int K, int dtype, hipStream_t s);
int launch_latent_gather(const void* cache, const int32_t* tables, int table_width, int block_size, const int32_t* k_begin,
                         const int32_t* k_lens, int n_seqs, int max_k, int row_elems, void* out, int dtype, hipStream_t s);

// ---- latent_prompt.hip ----
struct LatentPromptProblem {
    const uint16_t* q;       // rotated already
    int64_t q_stride;
    const uint16_t* k;       // [keys, heads * dim], sequence s from row k_begin[s]
    int64_t k_stride;
    const uint16_t* k_rot;
    int64_t k_rot_stride;
    const uint16_t* vt;      // [heads * vdim, keys]
    int64_t v_stride;
    uint16_t* out;           // [T, heads * vdim]
    const float* sink;
    const int32_t *q_begin, *starts, *k_begin;
    int heads, dim, rot, vdim;
    float scale;
};
bool latent_prompt_supported(int dim, int rot, int vdim);
int launch_latent_prompt(const LatentPromptProblem& p, int n_seqs, int max_q, hipStream_t s);

}  // namespace em
