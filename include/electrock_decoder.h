/*
 * electrock_decoder.h — C ABI of libelectrock_decoder.so (MI355X / gfx950): the kernels of decoders whose residual
 * stream is float32 (row kernels), of gated linear attention, of recurrences with one decay per head, and of latent and
 * softmax attention over a paged cache.
 *
 * Same conventions as electrock_moe.h: raw DEVICE pointers, plain sizes, a HIP stream passed as void*; asynchronous,
 * no allocation, no retained state; the device that owns the pointers is current.  Returns 0, an EM_ERR_* code (nothing
 * was launched) or a hipError_t.
 *
 * Element types: EM_DTYPE_BF16 or EM_DTYPE_F32 is the compute type `dtype` of activations, weights and key cache.
 * With EM_DTYPE_F32 every product is a float32 MFMA.  Pointers are aligned to 16 bytes unless said otherwise.
 */
#ifndef ELECTROCK_DECODER_H
#define ELECTROCK_DECODER_H

#include "electrock_moe.h"

#ifdef __cplusplus
extern "C" {
#endif

int ed_version(void);

/* x[t] = table[tokens[t]] * scale (float32 [T, W]); copy (may be null): the same, rounded to dtype, rows copy_stride
 * elements apart. */
int ed_embed(const int32_t* tokens, const void* table, double scale, float* x, void* copy, int64_t copy_stride,
             int64_t T, int W, int dtype, void* stream);

/* Update of the float32 stream x [T, W] by a sublayer's result y [T, W] (y_dtype; or its float32 partial sums
 * [y_parts, T, W]), then the next sublayer's input:
 *   update 0: x stays      1: x += y / sqrt(mean(y^2) + eps) * post_w      2: x = y + post_w (post_w may be null)
 *   out (may be null): next_w ? x / sqrt(mean(x^2) + eps) * next_w : x, rounded to dtype, rows out_stride apart.
 * post_w, next_w: float32 [W]. */
int ed_residual_norm(int update, float* x, const void* y, int y_dtype, int y_parts, const float* post_w,
                     const float* next_w, void* out, int64_t out_stride, int64_t T, int W, double eps, int dtype, void* stream);

/* u = max(u, 0)^2, n elements in place. */
int ed_relu_squared(void* u, int64_t n, int dtype, void* stream);

/* out [T, ff] = silu(u[t][c]) * u[t][ff + c]; u [T, 2 ff]. */
int ed_silu_gate(const void* u, void* out, int64_t T, int ff, int dtype, void* stream);

/* y = y * silu(z), RMS-normed in `parts` equal parts of a row, times w: in place, y [T, parts * size], rows of z z_stride
 * elements apart, w float32 [parts * size]. */
int ed_gated_norm(void* y, const void* z, int64_t z_stride, const float* w, int64_t T, int parts, int size, double eps, int dtype,
                  void* stream);

/* out = act(x w^T) for a decode batch, bf16 operands: x [T, K], w [N, K], T <= 64 (fewer for large
 * weights), K a multiple of 64; act 0: none,
 * 1: max(v, 0)^2, 2: w is [2 N, K], out = silu(x w_c) * (x w_(N + c)) in bf16.  splits > 1: out is float32 [splits, T, N], partial sums over K (no act).  ed_skinny_gemm_splits: how
 * many fill the chip, 0 if the shape is not taken. */
int ed_skinny_gemm_splits(int64_t T, int N, int K);
int ed_skinny_gemm(const void* x, const void* w, void* out, int out_dtype, int splits, int64_t T, int N, int K, int act,
                   void* stream);

/* g [T, dim] = gelu_tanh(x gate^T) * table[tokens[t]][column0 + c]; x [T, W], gate [dim, W]. */
int ed_token_gate(const void* x, const void* gate, const int32_t* tokens, const void* table, int64_t table_stride,
                  int column0, void* g, int64_t T, int W, int dim, int dtype, void* stream);

/* The end of a layer with a per-layer token input in one launch (bf16; W a multiple of 4, see
 * ed_token_side_supported):
 *   x += y / rms(y) * post_w;  g = gelu_tanh(gate x) * table[tokens[t]][column0 ...];  p = proj g;
 *   x += p / rms(p) * side_norm;  out = next_w ? x / rms(x) * next_w : x, rounded to bf16.
 * gate [dim, W], proj [W, dim]; rms(v) = sqrt(mean(v^2) + eps); norm weights float32. */
int ed_token_side_supported(int W, int dim);
int ed_token_side(float* x, const void* y, const float* post_w, const void* gate, const void* proj, const int32_t* tokens,
                  const void* table, int64_t table_stride, int column0, const float* side_norm, const float* next_w, void* out,
                  int64_t out_stride, int64_t T, int W, int dim, double eps, void* stream);

/*
 * Gated linear attention: S_t = diag(alpha_t) S_(t-1) + k_t v_t^T, o_t = S_t^T (q_scale q_t), alpha =
 * sigmoid(a2 a1_t + bias)^(1/tau); o is RMS-normed per head with norm_w, multiplied by silu(g), rounded to dtype.
 * q, k: head h at h * dim of a row; v, g: at h * vdim; all rows, and a1's, are `stride` elements apart.
 * a2: [heads * dim, rank], rows a2_stride apart.  dim, vdim <= 256, rank <= 512.
 * states: float32 [slots, heads, dim, vdim]; a sequence with starts[s] == 0 begins at zero, whatever its slot holds.
 */
typedef struct ed_gla_args {
    const void *q, *k, *v, *g, *a1;
    int64_t stride;
    const void* a2;
    const float* bias;
    const float* norm_w;
    void* out;                 /* [T, heads * vdim] */
    const int32_t *slots;      /* [n_seqs] */
    const int32_t *starts;     /* [n_seqs] position of the sequence's first token in this call */
    float* states;
    /* prompts only: */
    float* log_decay;          /* [T, heads * dim] scratch */
    const int32_t* chunks;     /* [n_chunks][4]: sequence, first row, tokens (<= chunk_tokens), unused */
    const int32_t* seq_chunks; /* [n_seqs + 1] first chunk of every sequence; chunks of a sequence are consecutive */
    float* chunk_states;       /* [n_chunks, heads, dim, vdim] scratch, null if every sequence has one chunk */
    float* chunk_decay;        /* [n_chunks, heads, dim] scratch, null likewise */
    int32_t n_seqs, n_chunks, chunk_tokens /* a multiple of 16 */;
    int32_t heads, dim, vdim, rank, a2_stride, dtype;
    float tau, q_scale, eps;
} ed_gla_args;

/* Portions of prompts: any number of tokens per sequence. */
int ed_gla_prefill(const ed_gla_args* a, void* stream);
/* One token per sequence: row s belongs to sequence s. */
int ed_gla_step(const ed_gla_args* a, void* stream);

/*
 * Recurrences with one decay per head and token, behind short causal convolutions:
 *   S <- g S;  u = beta (v - S^T k) (delta rule), or beta v (additive rule: beta_in is null);  S <- S + k u^T;  o = S^T q
 * with a float32 state S [dim, vdim] per head; query/key head of head h: h / (heads / kv_heads).
 * log g = -exp(a_log) softplus(decay_in + dt_bias).  Delta rule: beta = sigmoid(beta_in), and o is RMS-normed per head
 * with norm_w and multiplied by silu(gate).  Additive rule: beta is that softplus, and skip * v is added to o (skip may be
 * null).  q, k, v are silu(sum_j conv_w[., j] x_(t - taps + 1 + j) + conv_b) of the projections; with unit_eps > 0, q and k
 * are then divided by sqrt(sum of squares + unit_eps); q is multiplied by q_scale.
 * q, k: head g at g * dim of a row; v, gate: head h at h * vdim; decay_in, beta_in: column h; all rows `stride` elements
 * apart.  dim, vdim <= 256, taps <= 16.
 * ring: the last projections of every sequence, [slots, taps, channels] in the compute type, position p in row p % taps,
 * channels = q, k, v one behind the other, as in conv_w and conv_b.  A sequence with starts[s] == 0 begins with zeros,
 * whatever its slot holds.
 */
typedef struct ed_recur_args {
    const void *q, *k, *v, *decay_in, *beta_in, *gate;
    int64_t stride;
    const float *conv_w, *conv_b, *a_log, *dt_bias, *skip, *norm_w;
    void* ring;
    float* states;             /* [slots, heads, dim, vdim] */
    void* out;                 /* [T, heads * vdim] */
    const int32_t *slots, *starts; /* [n_seqs] */
    /* prompts only: */
    const int32_t *q_begin;    /* [n_seqs + 1] */
    const int32_t *chunks, *seq_chunks; /* as for ed_gla_prefill */
    float *q_rows, *k_rows;    /* [T, kv_heads, round_up(dim, 16)] scratch */
    void* v_rows;              /* [T, heads * vdim] scratch, compute type */
    float* rates;              /* [T, heads, 2] scratch */
    float* blocks;             /* [n_chunks, chunk_tokens / 16, heads, ed_recur_record(delta)] scratch */
    float* chunk_states;       /* [n_chunks, heads, dim, vdim] scratch, null if every sequence has one chunk */
    float* chunk_trans;        /* [n_chunks, heads, round_up(dim, 16)^2] (delta) or [n_chunks, heads] scratch, null likewise */
    int32_t n_seqs, n_chunks, chunk_tokens /* a multiple of 16 */;
    int32_t heads, kv_heads, dim, vdim, taps, dtype;
    float q_scale, unit_eps, eps;
} ed_recur_args;

int ed_recur_record(int delta);
/* Portions of prompts: any number of tokens per sequence. */
int ed_recur_prefill(const ed_recur_args* a, void* stream);
/* One token per sequence: row s belongs to sequence s. */
int ed_recur_step(const ed_recur_args* a, void* stream);

/*
 * Softmax attention over a paged cache, query head h on key/value head h / (heads / kv_heads).  A token's cache row holds
 * kv_heads keys of round_up(dim, 8) elements and behind them kv_heads values of round_up(vdim, 8) (ed_attn_row_elems in
 * all), zeros in the padding; key j of sequence s is row tables[s][j / block_size] * block_size + j % block_size.
 * dim, vdim <= 256, rot even and <= dim.
 */
typedef struct ed_attn_args {
    const void *q, *k, *v;     /* projections, rows `stride` apart, heads next to each other */
    int64_t stride;
    const void* v_first;       /* rows v_first_stride apart: v becomes (1 - *mix) v + *mix v_first; null with mix */
    int64_t v_first_stride;
    const float* mix;
    const float *q_norm, *k_norm; /* [dim] weights of the heads' RMS norms, or null */
    const float* inv_freq;     /* [rot / 2]: pair (2i, 2i + 1) of the first rot elements turns by position * inv_freq[i] */
    const int32_t *positions, *cache_rows; /* [T] */
    void* cache;
    void* q_rows;              /* [T, heads, round_up(dim, 8)] scratch: queries, normed and rotated */
    void* out;                 /* [T, heads * vdim] */
    const int32_t *q_begin, *starts, *tables; /* [n_seqs + 1], [n_seqs], [n_seqs, table_width] */
    float *part_o, *part_ml;   /* [T * heads, splits, vdim], [T * heads, splits, 2] scratch, unused if splits == 1 */
    int64_t T;
    int32_t n_seqs, max_q, table_width, block_size, splits;
    int32_t heads, kv_heads, dim, vdim, rot, window /* keys a query sees, itself included; 0: all */, dtype;
    float scale, softcap /* score = softcap tanh(score / softcap); 0: none */, eps;
} ed_attn_args;

int ed_attn_row_elems(int kv_heads, int dim, int vdim);
/* Norms, rotation and mixing: keys and values into the cache, queries into q_rows. */
int ed_attn_prepare(const ed_attn_args* a, void* stream);
/* Any portions; the keys of a row are shared out over `splits` (<= 64) workgroups. */
int ed_attn_paged(const ed_attn_args* a, void* stream);
/* Long portions, bf16: the same result (see ed_attn_prompt_supported). */
int ed_attn_prompt_supported(int dim, int vdim);
int ed_attn_prompt(const ed_attn_args* a, void* stream);

/*
 * Latent attention.  The cache holds, per token, round_up(rank, 8) elements of the normed latent and round_up(rot, 8) of
 * the rotated key part (ed_latent_row_elems of them), zeros in the padding; key j of sequence s is row
 * tables[s][j / block_size] * block_size + j % block_size.  rank <= 512, rot even and <= 128.
 */
typedef struct ed_latent_args {
    void* q;                   /* rows q_stride apart, head h at h * (dim + rot): [dim plain, rot rotated] */
    int64_t q_stride;
    const void* down;          /* rows down_stride apart: [rank latent, rot key part] */
    int64_t down_stride;
    const float* latent_w;     /* [rank] */
    const float* inv_freq;     /* [rot / 2] */
    const int32_t* positions;  /* [T] */
    const int32_t* cache_rows; /* [T] */
    void* cache;
    const void* q_latent;      /* [T, heads, round_up(rank, 8)] */
    void* out;                 /* the same shape */
    const float* sink;         /* [heads] */
    const int32_t* q_begin;    /* [n_seqs + 1] first row of every sequence */
    const int32_t* starts;     /* [n_seqs] position of that row's token */
    const int32_t* tables;     /* [n_seqs, table_width] */
    float* part_o;             /* [T * heads, splits, round_up(rank, 8)] scratch, unused if splits == 1 */
    float* part_ml;            /* [T * heads, splits, 2] scratch */
    int64_t T;
    int32_t n_seqs, max_q, table_width, block_size, splits;
    int32_t heads, dim, rot, rank, dtype;
    float scale, eps;
} ed_latent_args;

int ed_latent_row_elems(int rank, int rot);
/* Norm of the latent, rotation of the key part (both into the cache) and of q's rotated parts (in place). */
int ed_latent_prepare(const ed_latent_args* a, void* stream);
/* out = sum_j p_j c_j per row and head, p = softmax of (q_latent . c_j + q_rot . k_rot_j) * scale over the keys
 * j <= position with exp(sink) added to the denominator; the keys of a row are shared out over `splits` (<= 256) workgroups. */
int ed_latent_paged(const ed_latent_args* a, void* stream);
/* out[t, h, n] = sum_k a[t, h, k] b[h][n][k]; b: [heads, N, round_up(K, 32)], zeros in the padding. */
int ed_head_gemm(const void* a, int64_t a_row, int64_t a_head, const void* b, void* out, int64_t out_row,
                 int64_t out_head, int64_t T, int heads, int N, int K, int dtype, void* stream);
/* Cached rows of every sequence behind each other: out row k_begin[s] + j = key j of s, zeros from k_lens[s] on. */
int ed_latent_gather(const void* cache, const int32_t* tables, int table_width, int block_size,
                     const int32_t* k_begin, const int32_t* k_lens, int n_seqs, int max_k, int row_elems, void* out,
                     int dtype, void* stream);

/*
 * Latent attention of long portions with the keys and values written out (bf16 only): k [keys, heads * dim], the
 * transposed values vt [heads * vdim, keys] and the rotated key part k_rot, all for the whole context of every sequence,
 * sequence s from key k_begin[s].  Every k_begin is a multiple of 64 and the rows (columns of vt) from a sequence's last
 * key to the next multiple of 64 exist and are finite.  q is rotated already.  ed_latent_prompt_supported: which sizes.
 */
typedef struct ed_latent_prompt_args {
    const void* q;             /* rows q_stride apart, head h at h * (dim + rot) */
    int64_t q_stride;
    const void* k;
    int64_t k_stride;
    const void* k_rot;
    int64_t k_rot_stride;
    const void* vt;
    int64_t v_stride;
    void* out;                 /* [T, heads * vdim] */
    const float* sink;         /* [heads] */
    const int32_t *q_begin, *starts, *k_begin; /* [n_seqs + 1], [n_seqs], [n_seqs] */
    int32_t n_seqs, max_q, heads, dim, rot, vdim;
    float scale;               /* > 0 */
} ed_latent_prompt_args;

int ed_latent_prompt_supported(int dim, int rot, int vdim);
int ed_latent_prompt(const ed_latent_prompt_args* a, void* stream);

#ifdef __cplusplus
}
#endif
#endif
