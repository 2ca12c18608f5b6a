// extern "C" surface of libelectrock_decoder.so: argument checks and stage sequencing.
#include "decoder.h"

using namespace em;

namespace {

inline hipStream_t as_stream(void* s) { return static_cast<hipStream_t>(s); }
inline bool dtype_ok(int d) { return d == EM_DTYPE_F32 || d == EM_DTYPE_BF16; }
inline bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }
constexpr int64_t kMaxRows = 1 << 24;   // rows of one call: grids and 32-bit row numbers
constexpr int kMaxSeqs = 65535;

GlaProblem gla_problem(const ed_gla_args& a) {
    GlaProblem g;
    g.q = a.q; g.k = a.k; g.v = a.v; g.g = a.g; g.a1 = a.a1;
    g.stride = a.stride;
    g.a2 = a.a2; g.rank = a.rank; g.a2_stride = a.a2_stride;
    g.bias = a.bias; g.tau = a.tau;
    g.norm_w = a.norm_w; g.out = a.out;
    g.bl = a.log_decay; g.chunks = a.chunks;
    g.slots = a.slots; g.starts = a.starts;
    g.states = a.states; g.chunk_states = a.chunk_states; g.chunk_decay = a.chunk_decay;
    g.heads = a.heads; g.dim = a.dim; g.vdim = a.vdim;
    g.q_scale = a.q_scale; g.eps = a.eps; g.dtype = a.dtype;
    return g;
}

int check_gla(const ed_gla_args* a) {
    if (!a) return EM_ERR_NULL_POINTER;
    if (!dtype_ok(a->dtype)) return EM_ERR_BAD_DTYPE;
    if (a->n_seqs < 0 || a->n_seqs > kMaxSeqs || a->a2_stride < a->rank || !(a->tau > 0.0f)) return EM_ERR_BAD_SHAPE;
    if (!gla_supported(a->heads, a->dim, a->vdim, a->rank)) return EM_ERR_UNSUPPORTED;
    if (a->n_seqs == 0) return 0;
    if (!a->q || !a->k || !a->v || !a->g || !a->a1 || !a->a2 || !a->bias || !a->norm_w || !a->out || !a->slots ||
        !a->starts || !a->states)
        return EM_ERR_NULL_POINTER;
    if (!aligned16(a->states) || !aligned16(a->chunk_states) || !aligned16(a->a2)) return EM_ERR_ALIGNMENT;
    return 0;
}

LatentProblem latent_problem(const ed_latent_args& a) {
    LatentProblem p;
    p.q = a.q; p.q_stride = a.q_stride;
    p.down = a.down; p.down_stride = a.down_stride;
    p.latent_w = a.latent_w; p.inv_freq = a.inv_freq;
    p.positions = a.positions; p.cache_rows = a.cache_rows;
    p.cache = a.cache; p.q_latent = a.q_latent; p.out = a.out; p.sink = a.sink;
    p.q_begin = a.q_begin; p.starts = a.starts; p.tables = a.tables;
    p.table_width = a.table_width; p.block_size = a.block_size;
    p.heads = a.heads; p.dim = a.dim; p.rot = a.rot; p.rank = a.rank;
    p.scale = a.scale; p.eps = a.eps; p.dtype = a.dtype;
    return p;
}

int check_latent(const ed_latent_args* a) {
    if (!a) return EM_ERR_NULL_POINTER;
    if (!dtype_ok(a->dtype)) return EM_ERR_BAD_DTYPE;
    if (a->T < 0 || a->T > kMaxRows) return EM_ERR_BAD_SHAPE;
    if (!latent_supported(a->heads, a->dim, a->rot, a->rank)) return EM_ERR_UNSUPPORTED;
    return 0;
}

RecurProblem recur_problem(const ed_recur_args& a) {
    RecurProblem p;
    p.q = a.q; p.k = a.k; p.v = a.v;
    p.decay_in = a.decay_in; p.beta_in = a.beta_in; p.gate = a.gate;
    p.stride = a.stride;
    p.conv_w = a.conv_w; p.conv_b = a.conv_b;
    p.a_log = a.a_log; p.dt_bias = a.dt_bias; p.skip = a.skip; p.norm_w = a.norm_w;
    p.ring = a.ring; p.states = a.states; p.out = a.out;
    p.slots = a.slots; p.starts = a.starts; p.q_begin = a.q_begin;
    p.chunks = reinterpret_cast<const int4*>(a.chunks); p.seq_chunks = a.seq_chunks;
    p.q_f = a.q_rows; p.k_f = a.k_rows; p.v_f = a.v_rows;
    p.rates = a.rates; p.blocks = a.blocks; p.chunk_states = a.chunk_states; p.chunk_trans = a.chunk_trans;
    p.n_seqs = a.n_seqs; p.n_chunks = a.n_chunks; p.chunk_tokens = a.chunk_tokens;
    p.heads = a.heads; p.kv_heads = a.kv_heads; p.dim = a.dim; p.vdim = a.vdim; p.taps = a.taps; p.dtype = a.dtype;
    p.q_scale = a.q_scale; p.unit_eps = a.unit_eps; p.eps = a.eps;
    return p;
}

int check_recur(const ed_recur_args* a) {
    if (!a) return EM_ERR_NULL_POINTER;
    if (!dtype_ok(a->dtype)) return EM_ERR_BAD_DTYPE;
    if (a->n_seqs < 0 || a->n_seqs > kMaxSeqs) return EM_ERR_BAD_SHAPE;
    if (!recur_supported(a->heads, a->kv_heads, a->dim, a->vdim, a->taps)) return EM_ERR_UNSUPPORTED;
    if (a->n_seqs == 0) return 0;
    if (!a->q || !a->k || !a->v || !a->decay_in || (a->beta_in && (!a->gate || !a->norm_w)) || !a->conv_w || !a->a_log || !a->dt_bias ||
        !a->ring || !a->states || !a->out || !a->slots || !a->starts)
        return EM_ERR_NULL_POINTER;
    if (!aligned16(a->states) || !aligned16(a->ring) || !aligned16(a->conv_w)) return EM_ERR_ALIGNMENT;
    return 0;
}

AttnProblem attn_problem(const ed_attn_args& a) {
    AttnProblem p;
    p.q = a.q; p.k = a.k; p.v = a.v;
    p.stride = a.stride;
    p.v_first = a.v_first; p.v_first_stride = a.v_first_stride; p.mix = a.mix;
    p.q_norm = a.q_norm; p.k_norm = a.k_norm; p.inv_freq = a.inv_freq;
    p.positions = a.positions; p.cache_rows = a.cache_rows;
    p.cache = a.cache; p.q_out = a.q_rows; p.out = a.out;
    p.q_begin = a.q_begin; p.starts = a.starts; p.tables = a.tables;
    p.table_width = a.table_width; p.block_size = a.block_size;
    p.heads = a.heads; p.kv_heads = a.kv_heads; p.dim = a.dim; p.vdim = a.vdim; p.rot = a.rot; p.window = a.window; p.dtype = a.dtype;
    p.scale = a.scale; p.softcap = a.softcap; p.eps = a.eps;
    return p;
}

int check_attn(const ed_attn_args* a, bool attend) {
    if (!a) return EM_ERR_NULL_POINTER;
    if (!dtype_ok(a->dtype)) return EM_ERR_BAD_DTYPE;
    if (a->T < 0 || a->T > kMaxRows || a->window < 0 || !(a->softcap >= 0.0f)) return EM_ERR_BAD_SHAPE;
    if (!attn_supported(a->heads, a->kv_heads, a->dim, a->vdim, a->rot)) return EM_ERR_UNSUPPORTED;
    if (a->T == 0) return 0;
    if (!a->cache || !a->q_rows) return EM_ERR_NULL_POINTER;
    if (!aligned16(a->cache) || !aligned16(a->q_rows)) return EM_ERR_ALIGNMENT;
    if (!attend) return 0;
    if (a->n_seqs <= 0 || static_cast<int64_t>(a->n_seqs) * a->kv_heads > 65535 || a->max_q <= 0 || a->max_q > a->T || a->block_size <= 0 ||
        a->table_width <= 0)
        return EM_ERR_BAD_SHAPE;
    if (!a->out || !a->q_begin || !a->starts || !a->tables) return EM_ERR_NULL_POINTER;
    return 0;
}

}  // namespace

extern "C" {

int ed_version(void) { return 110; }

int ed_embed(const int32_t* tokens, const void* table, double scale, float* x, void* copy, int64_t copy_stride,
             int64_t T, int W, int dtype, void* stream) {
    if (!dtype_ok(dtype)) return EM_ERR_BAD_DTYPE;
    if (T < 0 || T > kMaxRows || !row_width_ok(W) || (copy && copy_stride < W)) return EM_ERR_BAD_SHAPE;
    if (T == 0) return 0;
    if (!tokens || !table || !x) return EM_ERR_NULL_POINTER;
    if (!aligned16(table) || !aligned16(x) || (W % 4 == 0 && (reinterpret_cast<uintptr_t>(copy) & 15) % (dtype == EM_DTYPE_F32 ? 16 : 8)))
        return EM_ERR_ALIGNMENT;
    return launch_embed(tokens, table, static_cast<float>(scale), x, copy, copy ? copy_stride : W, T, W, dtype, as_stream(stream));
}

int ed_residual_norm(int update, float* x, const void* y, int y_dtype, int y_parts, const float* post_w, const float* next_w,
                     void* out, int64_t out_stride, int64_t T, int W, double eps, int dtype, void* stream) {
    if (!dtype_ok(dtype) || (update != 0 && y_dtype != dtype && y_dtype != EM_DTYPE_F32)) return EM_ERR_BAD_DTYPE;
    if (y_parts < 1 || (y_parts > 1 && y_dtype != EM_DTYPE_F32)) return EM_ERR_BAD_SHAPE;
    if (update < 0 || update > 2 || T < 0 || T > kMaxRows || !row_width_ok(W) || (out && out_stride < W)) return EM_ERR_BAD_SHAPE;
    if (T == 0) return 0;
    if (!x || (update != 0 && !y) || (update == 1 && !post_w)) return EM_ERR_NULL_POINTER;
    // rows that are not a multiple of four elements go element by element
    if (W % 4 == 0 && (!aligned16(x) || !aligned16(y) || !aligned16(post_w) || !aligned16(next_w) || !aligned16(out)))
        return EM_ERR_ALIGNMENT;
    return launch_residual_norm(update, x, y, update == 0 ? dtype : y_dtype, y_parts, post_w, next_w, out, out ? out_stride : W, T, W,
                                static_cast<float>(eps), dtype, as_stream(stream));
}

int ed_relu_squared(void* u, int64_t n, int dtype, void* stream) {
    if (!dtype_ok(dtype)) return EM_ERR_BAD_DTYPE;
    if (n < 0 || n > (int64_t{1} << 38)) return EM_ERR_BAD_SHAPE;
    if (n == 0) return 0;
    if (!u) return EM_ERR_NULL_POINTER;
    if (!aligned16(u)) return EM_ERR_ALIGNMENT;
    return launch_relu_squared(u, n, dtype, as_stream(stream));
}

int ed_silu_gate(const void* u, void* out, int64_t T, int ff, int dtype, void* stream) {
    if (!dtype_ok(dtype)) return EM_ERR_BAD_DTYPE;
    if (T < 0 || T > kMaxRows || ff <= 0 || ff > (1 << 24)) return EM_ERR_BAD_SHAPE;
    if (T == 0) return 0;
    if (!u || !out) return EM_ERR_NULL_POINTER;
    if (!aligned16(u) || !aligned16(out)) return EM_ERR_ALIGNMENT;
    return launch_silu_gate(u, out, T, ff, dtype, as_stream(stream));
}

int ed_gated_norm(void* y, const void* z, int64_t z_stride, const float* w, int64_t T, int parts, int size, double eps, int dtype,
                  void* stream) {
    if (!dtype_ok(dtype)) return EM_ERR_BAD_DTYPE;
    if (T < 0 || T > kMaxRows || parts <= 0 || parts > 65535 || !row_width_ok(size) || z_stride < static_cast<int64_t>(parts) * size)
        return EM_ERR_BAD_SHAPE;
    if (T == 0) return 0;
    if (!y || !z || !w) return EM_ERR_NULL_POINTER;
    if (!aligned16(y) || !aligned16(z) || !aligned16(w)) return EM_ERR_ALIGNMENT;
    return launch_gated_norm(y, z, z_stride, w, T, parts, size, static_cast<float>(eps), dtype, as_stream(stream));
}

int ed_skinny_gemm_splits(int64_t T, int N, int K) { return skinny_supported(T, N, K) ? skinny_splits(static_cast<int>(T), N, K) : 0; }

int ed_skinny_gemm(const void* x, const void* w, void* out, int out_dtype, int splits, int64_t T, int N, int K, int act,
                   void* stream) {
    if (!dtype_ok(out_dtype)) return EM_ERR_BAD_DTYPE;
    if (T == 0) return 0;
    if (!skinny_supported(T, N, K)) return EM_ERR_UNSUPPORTED;
    if (splits < 1 || splits > 64 || splits > K / 64 || act < 0 || act > 2 ||
        (splits > 1 && (act != 0 || out_dtype != EM_DTYPE_F32)) || (act == 2 && out_dtype != EM_DTYPE_BF16))
        return EM_ERR_BAD_SHAPE;
    if (!x || !w || !out) return EM_ERR_NULL_POINTER;
    if (!aligned16(x) || !aligned16(w)) return EM_ERR_ALIGNMENT;
    return launch_skinny_gemm(x, w, out, out_dtype == EM_DTYPE_F32, splits, static_cast<int>(T), N, K, act, as_stream(stream));
}

int ed_token_gate(const void* x, const void* gate, const int32_t* tokens, const void* table, int64_t table_stride,
                  int column0, void* g, int64_t T, int W, int dim, int dtype, void* stream) {
    if (!dtype_ok(dtype)) return EM_ERR_BAD_DTYPE;
    if (T < 0 || T > kMaxRows || W <= 0 || dim <= 0 || dim > 16 * 65535 || column0 < 0 ||
        column0 + static_cast<int64_t>(dim) > table_stride)
        return EM_ERR_BAD_SHAPE;
    if (T == 0) return 0;
    if (!x || !gate || !tokens || !table || !g) return EM_ERR_NULL_POINTER;
    if (!aligned16(x) || !aligned16(gate)) return EM_ERR_ALIGNMENT;
    return launch_token_gate(x, gate, tokens, table, table_stride, column0, g, T, W, dim, dtype, as_stream(stream));
}

int ed_token_side_supported(int W, int dim) { return token_side_supported(W, dim) ? 1 : 0; }

int ed_token_side(float* x, const void* y, const float* post_w, const void* gate, const void* proj, const int32_t* tokens,
                  const void* table, int64_t table_stride, int column0, const float* side_norm, const float* next_w, void* out,
                  int64_t out_stride, int64_t T, int W, int dim, double eps, void* stream) {
    if (T < 0 || T > kMaxRows || column0 < 0 || column0 + static_cast<int64_t>(dim) > table_stride || out_stride < W) return EM_ERR_BAD_SHAPE;
    if (!token_side_supported(W, dim) || out_stride % 4 != 0) return EM_ERR_UNSUPPORTED;
    if (T == 0) return 0;
    if (!x || !y || !post_w || !gate || !proj || !tokens || !table || !side_norm || !out) return EM_ERR_NULL_POINTER;
    if (!aligned16(x) || !aligned16(y) || !aligned16(post_w) || !aligned16(gate) || !aligned16(proj) || !aligned16(side_norm) ||
        !aligned16(next_w) || !aligned16(out))
        return EM_ERR_ALIGNMENT;
    TokenSideProblem p{};
    p.x = x;
    p.y = static_cast<const uint16_t*>(y);
    p.post_w = post_w; p.side_norm = side_norm; p.next_w = next_w;
    p.gate = static_cast<const uint16_t*>(gate);
    p.proj = static_cast<const uint16_t*>(proj);
    p.tokens = tokens;
    p.table = static_cast<const uint16_t*>(table);
    p.table_stride = table_stride;
    p.column0 = column0;
    p.out = static_cast<uint16_t*>(out);
    p.out_stride = out_stride;
    p.T = T;
    p.W = W; p.dim = dim;
    p.eps = static_cast<float>(eps);
    return launch_token_side(p, as_stream(stream));
}

int ed_gla_prefill(const ed_gla_args* a, void* stream) {
    int rc = check_gla(a);
    if (rc != 0 || a->n_seqs == 0) return rc;
    if (a->n_chunks < a->n_seqs || a->chunk_tokens <= 0 || a->chunk_tokens % 16 != 0 || a->chunk_tokens / 16 > 65535) return EM_ERR_BAD_SHAPE;
    if (a->n_chunks > a->n_seqs && (!a->chunk_states || !a->chunk_decay)) return EM_ERR_WORKSPACE;
    if (!a->log_decay || !a->chunks || !a->seq_chunks) return EM_ERR_NULL_POINTER;
    if (!aligned16(a->chunks)) return EM_ERR_ALIGNMENT;
    GlaProblem g = gla_problem(*a);
    if (a->n_chunks == a->n_seqs) g.chunk_states = nullptr;
    return launch_gla_prefill(g, a->seq_chunks, a->n_chunks, a->n_seqs, a->chunk_tokens, as_stream(stream));
}

int ed_gla_step(const ed_gla_args* a, void* stream) {
    const int rc = check_gla(a);
    if (rc != 0 || a->n_seqs == 0) return rc;
    return launch_gla_step(gla_problem(*a), a->n_seqs, as_stream(stream));
}

int ed_recur_record(int delta) { return recur_record(delta != 0); }

int ed_recur_prefill(const ed_recur_args* a, void* stream) {
    const int rc = check_recur(a);
    if (rc != 0 || a->n_seqs == 0) return rc;
    if (a->n_chunks < a->n_seqs || a->chunk_tokens <= 0 || a->chunk_tokens % 16 != 0 || a->chunk_tokens / 16 > 65535) return EM_ERR_BAD_SHAPE;
    if (!a->q_rows || !a->k_rows || !a->v_rows || !a->rates || !a->blocks || (a->n_chunks > a->n_seqs && (!a->chunk_states || !a->chunk_trans)))
        return EM_ERR_WORKSPACE;
    if (!a->q_begin || !a->chunks || !a->seq_chunks) return EM_ERR_NULL_POINTER;
    if (!aligned16(a->chunks) || !aligned16(a->q_rows) || !aligned16(a->k_rows) || !aligned16(a->v_rows) || !aligned16(a->rates) ||
        !aligned16(a->blocks) || !aligned16(a->chunk_states) || !aligned16(a->chunk_trans))
        return EM_ERR_ALIGNMENT;
    RecurProblem p = recur_problem(*a);
    if (a->n_chunks == a->n_seqs) p.chunk_states = nullptr;
    return launch_recur_prefill(p, as_stream(stream));
}

int ed_recur_step(const ed_recur_args* a, void* stream) {
    const int rc = check_recur(a);
    if (rc != 0 || a->n_seqs == 0) return rc;
    return launch_recur_step(recur_problem(*a), as_stream(stream));
}

int ed_attn_row_elems(int kv_heads, int dim, int vdim) { return attn_row_elems(kv_heads, dim, vdim); }

int ed_attn_prepare(const ed_attn_args* a, void* stream) {
    const int rc = check_attn(a, false);
    if (rc != 0 || a->T == 0) return rc;
    if (!a->q || !a->k || !a->v || (a->mix && !a->v_first) || (a->rot > 0 && !a->inv_freq) || !a->positions || !a->cache_rows)
        return EM_ERR_NULL_POINTER;
    return launch_attn_prepare(attn_problem(*a), a->T, as_stream(stream));
}

int ed_attn_paged(const ed_attn_args* a, void* stream) {
    const int rc = check_attn(a, true);
    if (rc != 0 || a->T == 0) return rc;
    if (a->splits < 1 || a->splits > kAttnMaxSplits) return EM_ERR_BAD_SHAPE;
    if (a->splits > 1 && (!a->part_o || !a->part_ml)) return EM_ERR_WORKSPACE;
    return launch_attn_paged(attn_problem(*a), a->n_seqs, a->max_q, a->splits, a->part_o, a->part_ml, a->T, as_stream(stream));
}

int ed_attn_prompt_supported(int dim, int vdim) { return attn_prompt_supported(dim, vdim) ? 1 : 0; }

int ed_attn_prompt(const ed_attn_args* a, void* stream) {
    const int rc = check_attn(a, true);
    if (rc != 0 || a->T == 0) return rc;
    if (!attn_prompt_supported(a->dim, a->vdim) || a->dtype != EM_DTYPE_BF16 || a->max_q > 128 * 65535) return EM_ERR_UNSUPPORTED;
    if (!aligned16(a->out)) return EM_ERR_ALIGNMENT;
    return launch_attn_prompt(attn_problem(*a), a->n_seqs, a->max_q, as_stream(stream));
}

int ed_latent_row_elems(int rank, int rot) { return latent_row_elems(rank, rot); }

int ed_latent_prepare(const ed_latent_args* a, void* stream) {
    const int rc = check_latent(a);
    if (rc != 0 || a->T == 0) return rc;
    if (!a->q || !a->down || !a->latent_w || (a->rot > 0 && !a->inv_freq) || !a->positions || !a->cache_rows || !a->cache)
        return EM_ERR_NULL_POINTER;
    return launch_latent_prepare(latent_problem(*a), a->T, as_stream(stream));
}

int ed_latent_paged(const ed_latent_args* a, void* stream) {
    const int rc = check_latent(a);
    if (rc != 0 || a->T == 0) return rc;
    if (a->n_seqs <= 0 || a->n_seqs > kMaxSeqs || a->max_q <= 0 || a->max_q > a->T || a->splits < 1 || a->splits > kLatentMaxSplits ||
        a->block_size <= 0 || a->table_width <= 0)
        return EM_ERR_BAD_SHAPE;
    if (!a->q || !a->q_latent || !a->cache || !a->out || !a->sink || !a->q_begin || !a->starts || !a->tables) return EM_ERR_NULL_POINTER;
    if (a->splits > 1 && (!a->part_o || !a->part_ml)) return EM_ERR_WORKSPACE;
    if (!aligned16(a->cache) || !aligned16(a->q_latent)) return EM_ERR_ALIGNMENT;
    return launch_latent_paged(latent_problem(*a), a->n_seqs, a->max_q, a->splits, a->part_o, a->part_ml, a->T, as_stream(stream));
}

int ed_head_gemm(const void* a, int64_t a_row, int64_t a_head, const void* b, void* out, int64_t out_row,
                 int64_t out_head, int64_t T, int heads, int N, int K, int dtype, void* stream) {
    if (!dtype_ok(dtype)) return EM_ERR_BAD_DTYPE;
    if (T < 0 || T > kMaxRows || heads <= 0 || heads > 65535 || N <= 0 || K <= 0 || a_row < 0 || a_head < 0) return EM_ERR_BAD_SHAPE;
    if (T == 0) return 0;
    if (!a || !b || !out) return EM_ERR_NULL_POINTER;
    if (!aligned16(b)) return EM_ERR_ALIGNMENT;
    return launch_head_gemm(a, a_row, a_head, b, out, out_row, out_head, T, heads, N, K, dtype, as_stream(stream));
}

int ed_latent_gather(const void* cache, const int32_t* tables, int table_width, int block_size,
                     const int32_t* k_begin, const int32_t* k_lens, int n_seqs, int max_k, int row_elems, void* out,
                     int dtype, void* stream) {
    if (!dtype_ok(dtype)) return EM_ERR_BAD_DTYPE;
    if (n_seqs < 0 || n_seqs > kMaxSeqs || max_k < 0 || max_k > kMaxRows || row_elems <= 0 || row_elems % 8 != 0 ||
        block_size <= 0 || table_width <= 0)
        return EM_ERR_BAD_SHAPE;
    if (n_seqs == 0 || max_k == 0) return 0;
    if (!cache || !tables || !k_begin || !k_lens || !out) return EM_ERR_NULL_POINTER;
    if (!aligned16(cache) || !aligned16(out)) return EM_ERR_ALIGNMENT;
    return launch_latent_gather(cache, tables, table_width, block_size, k_begin, k_lens, n_seqs, max_k, row_elems, out, dtype,
                                as_stream(stream));
}

int ed_latent_prompt_supported(int dim, int rot, int vdim) { return latent_prompt_supported(dim, rot, vdim) ? 1 : 0; }

int ed_latent_prompt(const ed_latent_prompt_args* a, void* stream) {
    if (!a) return EM_ERR_NULL_POINTER;
    if (a->n_seqs < 0 || a->n_seqs > kMaxSeqs || a->max_q < 0 || a->max_q > kMaxRows || a->heads <= 0 || !(a->scale > 0.0f)) return EM_ERR_BAD_SHAPE;
    if (!latent_prompt_supported(a->dim, a->rot, a->vdim) || a->q_stride % 8 != 0 || a->k_stride % 8 != 0 ||
        a->k_rot_stride % 8 != 0 || a->v_stride % 8 != 0 || a->max_q > 128 * 65535)
        return EM_ERR_UNSUPPORTED;
    if (a->n_seqs == 0 || a->max_q == 0) return 0;
    if (!a->q || !a->k || (a->rot > 0 && !a->k_rot) || !a->vt || !a->out || !a->sink || !a->q_begin || !a->starts || !a->k_begin)
        return EM_ERR_NULL_POINTER;
    if (!aligned16(a->q) || !aligned16(a->k) || !aligned16(a->k_rot) || !aligned16(a->vt) || !aligned16(a->out)) return EM_ERR_ALIGNMENT;
    LatentPromptProblem p;
    p.q = static_cast<const uint16_t*>(a->q); p.q_stride = a->q_stride;
    p.k = static_cast<const uint16_t*>(a->k); p.k_stride = a->k_stride;
    p.k_rot = static_cast<const uint16_t*>(a->k_rot); p.k_rot_stride = a->k_rot_stride;
    p.vt = static_cast<const uint16_t*>(a->vt); p.v_stride = a->v_stride;
    p.out = static_cast<uint16_t*>(a->out);
    p.sink = a->sink;
    p.q_begin = a->q_begin; p.starts = a->starts; p.k_begin = a->k_begin;
    p.heads = a->heads; p.dim = a->dim; p.rot = a->rot; p.vdim = a->vdim;
    p.scale = a->scale;
    return launch_latent_prompt(p, a->n_seqs, a->max_q, as_stream(stream));
}

}  // extern "C"
