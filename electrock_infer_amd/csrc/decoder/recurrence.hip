// Recurrences with one decay per head and token, behind short causal convolutions:
//     S <- g S;   u = beta (v - S^T k)  (delta rule)   or   u = beta v  (additive rule);   S <- S + k u^T;   o = S^T q
// with a float32 state S [dim, vdim] per head and sequence; q and k are shared by heads / kv_heads heads.  The gated
// delta rule has beta = sigmoid(b) and unit vectors q and k, the state-space form has k = B, q = C, beta = dt and a skip
// o + D v; both have log g = -exp(A_log) softplus(a + dt_bias), where dt is that softplus.
//
// Convolutions.  q, k and v are sums over the last `taps` projections of a channel, then SiLU.  A sequence keeps its last
// projections in a ring of `taps` rows, position p in row p % taps: a step reads other rows than the one it writes, so
// that workgroups which share channels need no order among them.
//
// Prompts.  A sequence's tokens are cut into chunks and a chunk into blocks of 16.  With c_t the product of the decays
// from the block's first token to t and S the state in front of the block,
//     (I + A) U = diag(beta) (V - diag(c) K S),        A_ts = beta_t (c_t / c_s) k_t . k_s   for s < t   (0: additive)
//     o_t = c_t S^T q_t + sum_{s <= t} (c_t / c_s) (q_t . k_s) u_s
//     S  <- c_16 S + sum_s (c_16 / c_s) k_s u_s^T
// block_kernel makes (I + A)^-1 diag(beta) and the 16 x 16 scores of every block, all blocks in parallel.  chunk_kernel
// walks through the blocks of a chunk with float32 MFMAs, a wave holding 16 columns of the state in the registers in
// which an MFMA leaves them, which are the next MFMA's second operand as they are.  With several chunks in a sequence a
// first pass starts every chunk from zero, and for the delta rule, whose chunks multiply the state by a matrix, runs the
// identity's columns along, which gives that matrix; a scan over the chunks makes the states in front of them, and the
// output pass starts from there.  Ratios of decays are powers of differences of logarithms, never positive ones.
//
// Decoding.  One workgroup per (sequence, head): convolutions, decay, update, read-out, norm and gate; the state is read
// and written once.
#include <algorithm>

#include "decoder.h"

namespace em {
namespace {

constexpr int kBlock = 16;
constexpr float kLog2e = 1.4426950408889634f;
constexpr int kConvPiece = 256;      // channels of one wave of the convolution
constexpr int kMaxTaps = 16;

// A block's record, in floats: 16 x 16 scores, c_t, c_16 / c_t, beta_t, log2 of c_16 (16 of them); delta rule: the inverse
constexpr int kRecScores = 0, kRecDecay = 256, kRecRest = 272, kRecBeta = 288, kRecLog = 304, kRecInverse = 320;
static_assert(recur_record(false) == kRecInverse && recur_record(true) == kRecInverse + 256, "a block's record");

__device__ __forceinline__ float exp2_fast(float x) { return __builtin_amdgcn_exp2f(x); }
// with the hardware's exponential, reciprocal and square root, 1 ulp each
__device__ __forceinline__ float silu_fast(float g) { return g * __builtin_amdgcn_rcpf(1.0f + exp2_fast(-g * kLog2e)); }
__device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int off = kWave / 2; off > 0; off >>= 1) v += __shfl_xor(v, off);
    return v;
}

// log2 of the decay, and beta (dt for the additive rule)
template <typename Elem>
__device__ __forceinline__ f32x2_t decay_and_beta(const RecurProblem& p, int64_t row, int h) {
    typedef typename Elem::storage S;
    const float sp = softplus(Elem::load(static_cast<const S*>(p.decay_in)[row * p.stride + h]) + p.dt_bias[h]);
    const float log_g = -expf(p.a_log[h]) * sp * kLog2e;
    return f32x2_t{log_g, p.beta_in ? sigmoid(Elem::load(static_cast<const S*>(p.beta_in)[row * p.stride + h])) : sp};
}

template <typename Elem, bool VEC>
__device__ __forceinline__ void load_channels(const typename Elem::storage* src, int c, int count, float (&v)[4]) {
    if (VEC) {
        if (c < count) {
            typename Elem::storage t[4];
            __builtin_memcpy(t, __builtin_assume_aligned(src + c, sizeof(t)), sizeof(t));
#pragma unroll
            for (int j = 0; j < 4; ++j) v[j] = Elem::load(t[j]);
        } else {
#pragma unroll
            for (int j = 0; j < 4; ++j) v[j] = 0.0f;
        }
    } else {
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = c + j < count ? Elem::load(src[c + j]) : 0.0f;
    }
}

// ---- prompts: convolutions, unit vectors, decays ----
// A wave takes 16 tokens of kConvPiece channels: four per lane, of as many q or k heads as fit (a head has a power of two of
// lanes, `head_lanes`) or of v; the last waves' share is decays and betas, one per lane.  K >= taps: rows that a lane keeps.  VEC: all
// counts and offsets are multiples of four.
template <typename Elem, int K, bool VEC>
__global__ __launch_bounds__(256) void recur_conv_kernel(RecurProblem p, int head_lanes) {
    typedef typename Elem::storage S;
    const int4 ch = p.chunks[blockIdx.x];
    const int first = blockIdx.y * kBlock;
    if (first >= ch.z) return;
    const int n = min(kBlock, ch.z - first), seq = ch.x;
    const int64_t row0 = static_cast<int64_t>(ch.y) + first;
    const int q_begin = p.q_begin[seq], n_seq = p.q_begin[seq + 1] - q_begin;
    const int at0 = static_cast<int>(row0) - q_begin;          // in this step's portion of the sequence
    const int start = p.starts[seq], pos0 = start + at0;
    const int lane = threadIdx.x & 63;
    const int v_count = p.heads * p.vdim, v_units = (v_count + kConvPiece - 1) / kConvPiece;
    const int fit = kWave / head_lanes, head_units = (p.kv_heads + fit - 1) / fit;
    const int unit = blockIdx.z * 4 + (threadIdx.x >> 6);
    if (unit >= 2 * head_units + v_units) {
        const int i = (unit - 2 * head_units - v_units) * kWave + lane, t = i / p.heads, h = i - t * p.heads;
        if (t < n) *reinterpret_cast<f32x2_t*>(p.rates + ((row0 + t) * p.heads + h) * 2) = decay_and_beta<Elem>(p, row0 + t, h);
        return;
    }
    const bool is_v = unit >= 2 * head_units, is_q = unit < head_units;
    const int g = is_v ? 0 : (is_q ? unit : unit - head_units) * fit + lane / head_lanes;      // this lane's q or k head
    const int begin = is_v ? (unit - 2 * head_units) * kConvPiece : g * p.dim;
    const int count = is_v ? min(kConvPiece, v_count - begin) : g < p.kv_heads ? p.dim : 0;
    const S* src = static_cast<const S*>(is_v ? p.v : is_q ? p.q : p.k) + begin;
    const int c = (is_v ? lane : lane % head_lanes) * 4;
    const int channels = 2 * p.kv_heads * p.dim + v_count;
    const int channel0 = (is_v ? 2 * p.kv_heads * p.dim : is_q ? 0 : p.kv_heads * p.dim) + begin;
    S* ring = static_cast<S*>(p.ring) + static_cast<int64_t>(p.slots[seq]) * p.taps * channels + channel0;

    float cur[kBlock][4];
#pragma unroll
    for (int t = 0; t < kBlock; ++t) load_channels<Elem, VEC>(src + (row0 + min(t, n - 1)) * p.stride, c, count, cur[t]);
    float w[K][4], bias[4];                                     // w[i]: of the row K - 1 - i tokens back
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        bias[j] = p.conv_b != nullptr && c + j < count ? p.conv_b[channel0 + c + j] : 0.0f;
        if (K == 4 && p.taps == 4) {
            f32x4_t row = {0.0f, 0.0f, 0.0f, 0.0f};
            if (c + j < count) row = *reinterpret_cast<const f32x4_t*>(p.conv_w + static_cast<int64_t>(channel0 + c + j) * 4);
#pragma unroll
            for (int i = 0; i < K; ++i) w[i][j] = row[i & 3];
            continue;
        }
#pragma unroll
        for (int i = 0; i < K; ++i)
            w[i][j] = K - 1 - i < p.taps && c + j < count ? p.conv_w[static_cast<int64_t>(channel0 + c + j) * p.taps + p.taps - K + i] : 0.0f;
    }
    float hist[K][4];                                           // hist[i]: the row K - 1 - i back, hist[K - 1] unused
#pragma unroll
    for (int i = 0; i < K; ++i) {
        const int back = K - 1 - i;
#pragma unroll
        for (int j = 0; j < 4; ++j) hist[i][j] = 0.0f;
        if (back > 0 && back < p.taps) {
            if (at0 >= back) load_channels<Elem, VEC>(src + (row0 - back) * p.stride, c, count, hist[i]);
            else if (pos0 >= back) load_channels<Elem, VEC>(ring + static_cast<int64_t>((pos0 - back) % p.taps) * channels, c, count, hist[i]);
        }
    }
    const int dp = (p.dim + 15) / 16 * 16;
#pragma unroll
    for (int t = 0; t < kBlock; ++t) {
        float y[4], ss = 0.0f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            y[j] = bias[j];
#pragma unroll
            for (int i = 0; i < K - 1; ++i) {
                y[j] = fmaf(w[i][j], hist[i][j], y[j]);
                hist[i][j] = i + 1 < K - 1 ? hist[i + 1][j] : cur[t][j];
            }
            y[j] = silu_fast(fmaf(w[K - 1][j], cur[t][j], y[j]));
            ss = fmaf(y[j], y[j], ss);
        }
        const int64_t row = row0 + t;
        if (is_v) {
            S* dst = static_cast<S*>(p.v_f) + row * v_count + begin;
            if (VEC) {
                if (c < count && t < n) {
                    S s4[4];
#pragma unroll
                    for (int j = 0; j < 4; ++j) s4[j] = Elem::store(y[j]);
                    __builtin_memcpy(__builtin_assume_aligned(dst + c, sizeof(s4)), s4, sizeof(s4));
                }
            } else {
#pragma unroll
                for (int j = 0; j < 4; ++j)
                    if (c + j < count && t < n) dst[c + j] = Elem::store(y[j]);
            }
        } else {
            float scale = is_q ? p.q_scale : 1.0f;
            if (p.unit_eps > 0.0f) {
                for (int off = head_lanes / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off);
                scale *= __builtin_amdgcn_rsqf(ss + p.unit_eps);
            }
            // (channels beyond dim are zero: their weights are)
            float* dst = (is_q ? p.q_f : p.k_f) + (row * p.kv_heads + g) * dp;
            if (c < dp && count > 0 && t < n) *reinterpret_cast<f32x4_t*>(dst + c) = f32x4_t{y[0] * scale, y[1] * scale, y[2] * scale, y[3] * scale};
        }
    }
    if (at0 != 0) return;
    // (the lane that reads the ring's old rows of these channels is the one that replaces them)
    S last[K][4];
#pragma unroll
    for (int back = 1; back < K; ++back)
#pragma unroll
        for (int j = 0; j < 4; ++j)
            last[back][j] = back < p.taps && back <= n_seq && c + j < count ? src[(static_cast<int64_t>(q_begin) + n_seq - back) * p.stride + c + j] : S(0);
#pragma unroll
    for (int back = 1; back < K; ++back) {
        if (back >= p.taps || back > n_seq) continue;
        S* dst = ring + static_cast<int64_t>((start + n_seq - back) % p.taps) * channels;
#pragma unroll
        for (int j = 0; j < 4; ++j)
            if (c + j < count) dst[c + j] = last[back][j];
    }
}

// ---- prompts: every block's scores and inverse ----
// A wave takes one block and up to kBlockHeads of the heads that share q and k.
constexpr int kBlockHeads = 8;
template <bool DELTA>
__global__ __launch_bounds__(256) void recur_block_kernel(RecurProblem p, int heads_per_wave) {
    constexpr int kPitch = 20;
    __shared__ __attribute__((aligned(16))) float lds[4][kBlock * kPitch];
    const int4 ch = p.chunks[blockIdx.x];
    const int first = blockIdx.y * kBlock;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, l16 = lane & 15, lq = lane >> 4;
    const int share = p.heads / p.kv_heads, h0 = (blockIdx.z * 4 + wave) * heads_per_wave;   // (a divisor of `share`)
    if (first >= ch.z || h0 >= p.heads) return;                 // (waves share nothing)
    const int n = min(kBlock, ch.z - first);
    const int64_t row0 = static_cast<int64_t>(ch.y) + first;
    const int dp = (p.dim + 15) / 16 * 16, g = h0 / share;
    const int64_t pitch = static_cast<int64_t>(p.kv_heads) * dp;
    const bool ok = l16 < n;
    const float* kr = p.k_f + (row0 + (ok ? l16 : 0)) * pitch + g * dp + lq * 4;
    const float* qr = p.q_f + (row0 + (ok ? l16 : 0)) * pitch + g * dp + lq * 4;
    f32x4_t qk = {0.0f, 0.0f, 0.0f, 0.0f}, kk = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll 4
    for (int d = 0; d < dp; d += 16) {
        const f32x4_t q4 = *reinterpret_cast<const f32x4_t*>(qr + d), k4 = *reinterpret_cast<const f32x4_t*>(kr + d);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            qk = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[r], k4[r], qk, 0, 0, 0);
            if (DELTA) kk = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[r], k4[r], kk, 0, 0, 0);
        }
    }
    const int64_t nb = p.chunk_tokens / kBlock;
    float* am = lds[wave];
    for (int h = h0; h < h0 + heads_per_wave; ++h) {
        f32x2_t rate = {0.0f, 0.0f};
        if (ok) rate = *reinterpret_cast<const f32x2_t*>(p.rates + ((row0 + l16) * p.heads + h) * 2);
        float bl = rate[0];
#pragma unroll
        for (int off = 1; off < kBlock; off <<= 1) {
            const float up = __shfl_up(bl, off, kBlock);
            if (l16 >= off) bl += up;
        }
        const float tot = __shfl(bl, kBlock - 1, kBlock);
        float* rec = p.blocks + ((blockIdx.x * nb + blockIdx.y) * p.heads + h) * recur_record(DELTA);
        if (lq == 0) {
            rec[kRecDecay + l16] = exp2_fast(bl);
            rec[kRecRest + l16] = exp2_fast(tot - bl);
            rec[kRecBeta + l16] = rate[1];
            rec[kRecLog + l16] = tot;
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = lq * 4 + r;
            const float ratio = exp2_fast(fminf(__shfl(bl, t, kBlock) - bl, 0.0f)), beta = __shfl(rate[1], t, kBlock);
            rec[kRecScores + t * kBlock + l16] = l16 <= t && t < n ? qk[r] * ratio : 0.0f;
            if (DELTA) am[t * kPitch + l16] = l16 < t && t < n ? beta * kk[r] * ratio : 0.0f;
        }
        if (!DELTA) continue;
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
        // column l16 of the inverse of the unit lower triangular matrix, row by row (each quarter of the wave on its own)
        float inv[kBlock];
#pragma unroll
        for (int t = 0; t < kBlock; ++t) {
            float v = t == l16 ? 1.0f : 0.0f;
#pragma unroll
            for (int s0 = 0; s0 < t; s0 += 4) {
                const f32x4_t a = *reinterpret_cast<const f32x4_t*>(am + t * kPitch + s0);
#pragma unroll
                for (int j = 0; j < 4; ++j)
                    if (s0 + j < t) v = fmaf(-a[j], inv[s0 + j], v);
            }
            inv[t] = v;
        }
#pragma unroll
        for (int t = 0; t < kBlock; ++t)
            if ((t >> 2) == lq) rec[kRecInverse + t * kBlock + l16] = inv[t] * rate[1];
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    }
}

// ---- prompts: a chunk's blocks, one after the other ----
// One workgroup per (chunk, head, group of column tiles), one wave per tile of 16 state columns; waves without a tile help
// with the loads.  OUTPUT: from the state in front of the chunk; else from zero, with the identity's columns behind the
// state's for the delta rule.
template <typename Elem, int NDT, bool DELTA, bool OUTPUT, int THREADS>
__global__ __launch_bounds__(THREADS) void recur_chunk_kernel(RecurProblem p) {
    typedef typename Elem::storage S;
    constexpr int D = NDT * 16, DP = D + 4, kPieces = (NDT + 3) / 4;   // four-float pieces of a block's k (q) per thread
    constexpr int kTile = kBlock * DP;
    const int waves = blockDim.x / kWave;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float* Ks = lds;                                  // [2][16][DP]
    float* Qs = Ks + 2 * kTile;                       // [2][16][DP]
    float* Rs = Qs + (OUTPUT ? 2 * kTile : 0);        // [2][waves][16] partial sums of squares

    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lq = lane >> 4;
    const int4 ch = p.chunks[blockIdx.x];
    const int h = blockIdx.y, dim = p.dim, vdim = p.vdim, dp = (dim + 15) / 16 * 16;
    const int g = h / (p.heads / p.kv_heads);
    const int v_tiles = (vdim + 15) / 16, tile = blockIdx.z * waves + wave;
    const bool identity = !OUTPUT && DELTA && tile >= v_tiles;
    const bool has_tile = tile < v_tiles || (identity && tile < v_tiles + dp / 16);
    const int col = (identity ? tile - v_tiles : tile) * 16 + l16;
    const bool v_ok = tile < v_tiles && col < vdim;
    const int64_t kq_pitch = static_cast<int64_t>(p.kv_heads) * dp, v_pitch = static_cast<int64_t>(p.heads) * vdim;
    const float* kg = p.k_f + g * dp;
    const float* qg = p.q_f + g * dp;
    const S* vg = static_cast<const S*>(p.v_f) + h * vdim + col;
    const S* gate = OUTPUT && DELTA ? static_cast<const S*>(p.gate) + h * vdim + col : nullptr;
    const int n_blocks = (ch.z + kBlock - 1) / kBlock;
    const int64_t rec_pitch = static_cast<int64_t>(p.heads) * recur_record(DELTA);
    const float* rec0 = p.blocks + (static_cast<int64_t>(blockIdx.x) * (p.chunk_tokens / kBlock) * p.heads + h) * recur_record(DELTA);

    f32x4_t st[NDT];                                  // rows dt * 16 + lq * 4 + r, column `col`
    const int64_t head_state = static_cast<int64_t>(dim) * vdim;
    float* slot = p.states + (static_cast<int64_t>(p.slots[ch.x]) * p.heads + h) * head_state;
    const bool chunked = p.chunk_states != nullptr;
    float* mine = chunked ? p.chunk_states + (static_cast<int64_t>(blockIdx.x) * p.heads + h) * head_state : slot;
    const bool from_zero = !OUTPUT || (!chunked && p.starts[ch.x] == 0);
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int d = dt * 16 + lq * 4 + r;
            st[dt][r] = identity ? (d == col ? 1.0f : 0.0f) : (!from_zero && v_ok && d < dim) ? mine[static_cast<int64_t>(d) * vdim + col] : 0.0f;
        }
    const float norm_w = OUTPUT && DELTA && v_ok ? p.norm_w[col] : 0.0f;
    const float skip = OUTPUT && p.skip != nullptr ? p.skip[h] : 0.0f;
    const float inv_vdim = 1.0f / static_cast<float>(vdim);

    // a block's operands, in flight while the one before is computed
    f32x4_t rk[kPieces], rq[kPieces], scores, inverse, decay, rest, beta;
    float block_decay, block_log;
    S v[4], gt[4];                                    // (as stored: a conversion here would wait for the load)
    auto fetch = [&](int b) {
        const int n = min(kBlock, ch.z - b * kBlock);
        const int64_t row0 = static_cast<int64_t>(ch.y) + b * kBlock;
#pragma unroll
        for (int i = 0; i < kPieces; ++i) {
            const int e = tid + i * static_cast<int>(blockDim.x), t = e / (D / 4), d = (e - t * (D / 4)) * 4;
            rk[i] = rq[i] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
            if (t < n && d < dp) {
                rk[i] = *reinterpret_cast<const f32x4_t*>(kg + (row0 + t) * kq_pitch + d);
                if (OUTPUT) rq[i] = *reinterpret_cast<const f32x4_t*>(qg + (row0 + t) * kq_pitch + d);
            }
        }
        const float* rec = rec0 + b * rec_pitch;
        if (OUTPUT) scores = *reinterpret_cast<const f32x4_t*>(rec + kRecScores + l16 * kBlock + lq * 4);
        if (DELTA) inverse = *reinterpret_cast<const f32x4_t*>(rec + kRecInverse + l16 * kBlock + lq * 4);
        else beta = *reinterpret_cast<const f32x4_t*>(rec + kRecBeta + lq * 4);
        decay = *reinterpret_cast<const f32x4_t*>(rec + kRecDecay + lq * 4);
        rest = *reinterpret_cast<const f32x4_t*>(rec + kRecRest + lq * 4);
        block_decay = rec[kRecDecay + kBlock - 1];
        block_log = rec[kRecLog];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = lq * 4 + r;
            const bool ok = v_ok && t < n;
            v[r] = ok ? vg[(row0 + t) * v_pitch] : S(0);
            if (OUTPUT && DELTA) gt[r] = ok ? gate[(row0 + t) * p.stride] : S(0);
        }
    };
    // a block's results wait for the row sums of the other waves until the next barrier
    f32x4_t held = {0.0f, 0.0f, 0.0f, 0.0f};
    float held_gate[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    auto finish = [&](int b) {
        const int n = min(kBlock, ch.z - b * kBlock);
        const int64_t row0 = static_cast<int64_t>(ch.y) + b * kBlock;
        f32x4_t ss = {0.0f, 0.0f, 0.0f, 0.0f};
        for (int w = 0; w < waves; ++w) ss += *reinterpret_cast<const f32x4_t*>(Rs + ((b & 1) * waves + w) * kBlock + lq * 4);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = lq * 4 + r;
            if (v_ok && t < n) {
                const float y = held[r] * __builtin_amdgcn_rsqf(ss[r] * inv_vdim + p.eps) * norm_w;
                static_cast<S*>(p.out)[(row0 + t) * v_pitch + h * vdim + col] = Elem::store(y * silu_fast(held_gate[r]));
            }
        }
    };
    float log_sum = 0.0f;
    fetch(0);
    for (int b = 0; b < n_blocks; ++b) {
        float* kb = Ks + (b & 1) * kTile;
        float* qb = Qs + (b & 1) * kTile;
#pragma unroll
        for (int i = 0; i < kPieces; ++i) {
            const int e = tid + i * static_cast<int>(blockDim.x), t = e / (D / 4), d = (e - t * (D / 4)) * 4;
            if (t < kBlock) {
                *reinterpret_cast<f32x4_t*>(kb + t * DP + d) = rk[i];
                if (OUTPUT) *reinterpret_cast<f32x4_t*>(qb + t * DP + d) = rq[i];
            }
        }
        const f32x4_t scores_b = scores, inverse_b = inverse, decay_b = decay, rest_b = rest, beta_b = beta;
        const float whole = block_decay;
        float v_b[4], gt_b[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            v_b[r] = Elem::load(v[r]);
            gt_b[r] = OUTPUT && DELTA ? Elem::load(gt[r]) : 0.0f;
        }
        log_sum += block_log;
        __syncthreads();              // (the block before last, in the same half, has been used)
        if (b + 1 < n_blocks) fetch(b + 1);
        if (OUTPUT && DELTA && b > 0) finish(b - 1);
        if (!has_tile) {
            if (OUTPUT && DELTA && lane < kBlock) Rs[((b & 1) * waves + wave) * kBlock + lane] = 0.0f;
            continue;
        }
        f32x4_t u;
        if (DELTA) {
            f32x4_t ks = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int dt = 0; dt < NDT; ++dt) {
                const f32x4_t k4 = *reinterpret_cast<const f32x4_t*>(kb + l16 * DP + dt * 16 + lq * 4);
#pragma unroll
                for (int r = 0; r < 4; ++r) ks = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[r], st[dt][r], ks, 0, 0, 0);
            }
            f32x4_t right;
#pragma unroll
            for (int r = 0; r < 4; ++r) right[r] = v_b[r] - decay_b[r] * ks[r];
            u = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int r = 0; r < 4; ++r) u = __builtin_amdgcn_mfma_f32_16x16x4f32(inverse_b[r], right[r], u, 0, 0, 0);
        } else {
#pragma unroll
            for (int r = 0; r < 4; ++r) u[r] = beta_b[r] * v_b[r];
        }
        if (OUTPUT) {
            f32x4_t o = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int dt = 0; dt < NDT; ++dt) {
                const f32x4_t q4 = *reinterpret_cast<const f32x4_t*>(qb + l16 * DP + dt * 16 + lq * 4);
#pragma unroll
                for (int r = 0; r < 4; ++r) o = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[r], st[dt][r], o, 0, 0, 0);
            }
            o *= decay_b;
#pragma unroll
            for (int r = 0; r < 4; ++r) o = __builtin_amdgcn_mfma_f32_16x16x4f32(scores_b[r], u[r], o, 0, 0, 0);
            if (DELTA) {
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    float ss = o[r] * o[r];
#pragma unroll
                    for (int off = 8; off > 0; off >>= 1) ss += __shfl_xor(ss, off);
                    if (l16 == 0) Rs[((b & 1) * waves + wave) * kBlock + lq * 4 + r] = ss;
                    held_gate[r] = gt_b[r];
                }
                held = o;
            } else {
                const int n = min(kBlock, ch.z - b * kBlock);
                const int64_t row0 = static_cast<int64_t>(ch.y) + b * kBlock;
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int t = lq * 4 + r;
                    if (v_ok && t < n)
                        static_cast<S*>(p.out)[(row0 + t) * v_pitch + h * vdim + col] = Elem::store(fmaf(skip, v_b[r], o[r]));
                }
            }
        }
        u *= rest_b;
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) {
            st[dt] *= whole;
            const float* kc = kb + lq * 4 * DP + dt * 16 + l16;
#pragma unroll
            for (int r = 0; r < 4; ++r) st[dt] = __builtin_amdgcn_mfma_f32_16x16x4f32(kc[r * DP], u[r], st[dt], 0, 0, 0);
        }
    }
    if (OUTPUT && DELTA) {
        __syncthreads();
        finish(n_blocks - 1);
    }
    if (OUTPUT && chunked) return;
    if (identity) {
        float* m = p.chunk_trans + (static_cast<int64_t>(blockIdx.x) * p.heads + h) * dp * dp;
        if (has_tile) {
#pragma unroll
            for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int d = dt * 16 + lq * 4 + r;
                    if (d < dp) m[d * dp + col] = st[dt][r];
                }
        }
        return;
    }
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int d = dt * 16 + lq * 4 + r;
            if (v_ok && d < dim) mine[static_cast<int64_t>(d) * vdim + col] = st[dt][r];
        }
    if (!OUTPUT && !DELTA && tile == 0 && lane == 0) p.chunk_trans[static_cast<int64_t>(blockIdx.x) * p.heads + h] = log_sum;
}

// ---- prompts: contribution of every chunk -> state in front of it; the state behind the last chunk goes to the slot ----
// Additive rule: a chunk multiplies the state by a number.
__global__ __launch_bounds__(256) void recur_scan_kernel(RecurProblem p) {
    constexpr int kAhead = 4;
    const int i = blockIdx.x * 256 + threadIdx.x, n = p.dim * p.vdim;
    if (i >= n) return;
    const int h = blockIdx.y, s = blockIdx.z;
    const int c0 = p.seq_chunks[s], c1 = p.seq_chunks[s + 1];
    const int64_t pitch = static_cast<int64_t>(p.heads) * n;
    float* slot = p.states + (static_cast<int64_t>(p.slots[s]) * p.heads + h) * n + i;
    float* cs = p.chunk_states + static_cast<int64_t>(h) * n + i;
    float state = p.starts[s] == 0 ? 0.0f : *slot;
    for (int c = c0; c < c1; c += kAhead) {
        float u[kAhead], e[kAhead];
#pragma unroll
        for (int j = 0; j < kAhead; ++j)
            if (c + j < c1) {
                u[j] = cs[(c + j) * pitch];
                e[j] = p.chunk_trans[static_cast<int64_t>(c + j) * p.heads + h];
            }
#pragma unroll
        for (int j = 0; j < kAhead; ++j)
            if (c + j < c1) {
                cs[(c + j) * pitch] = state;
                state = fmaf(exp2_fast(e[j]), state, u[j]);
            }
    }
    *slot = state;
}

// Delta rule: by a matrix.  One workgroup per (head, 16 state columns, sequence), one wave per 16 rows.
template <int NDT>
__global__ __launch_bounds__(NDT * kWave) void recur_matrix_scan_kernel(RecurProblem p) {
    constexpr int kPitch = NDT * 16 + 4;
    __shared__ __attribute__((aligned(16))) float state[2][16 * kPitch];      // column by column
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, lq = lane >> 4;
    const int col = blockIdx.y * 16 + l16, h = blockIdx.x, s = blockIdx.z;   // (a head's workgroups share an L2)
    const int dim = p.dim, vdim = p.vdim, dp = (dim + 15) / 16 * 16;
    const int c0 = p.seq_chunks[s], c1 = p.seq_chunks[s + 1];
    const int64_t n = static_cast<int64_t>(dim) * vdim, pitch = static_cast<int64_t>(p.heads) * n;
    const int64_t m_size = static_cast<int64_t>(dp) * dp, m_pitch = static_cast<int64_t>(p.heads) * m_size;
    float* slot = p.states + (static_cast<int64_t>(p.slots[s]) * p.heads + h) * n;
    float* cs = p.chunk_states + static_cast<int64_t>(h) * n;
    const int row = wave * 16 + lq * 4, k_tiles = dp / 16;
    const bool has_rows = wave * 16 < dp, zero = p.starts[s] == 0;
    const float* mr = p.chunk_trans + h * m_size + static_cast<int64_t>(has_rows ? wave * 16 + l16 : 0) * dp + lq * 4;
    // a chunk's matrix and contribution, in flight two chunks ahead (one, where the registers do not hold three matrices)
    constexpr int kAhead = NDT <= 8 ? 2 : 1;
    bool ok[4];
    f32x4_t cur, add[kAhead], m4[kAhead][NDT];
    // (addresses are held inside instead of loads being skipped: waits can count straight-line loads)
    int64_t from[4];
    auto fetch = [&](int c, f32x4_t& to_add, f32x4_t (&to)[NDT]) {
        c = min(c, c1 - 1);
#pragma unroll
        for (int r = 0; r < 4; ++r) to_add[r] = cs[c * pitch + from[r]];
#pragma unroll
        for (int k = 0; k < NDT; ++k) to[k] = *reinterpret_cast<const f32x4_t*>(mr + c * m_pitch + min(k, k_tiles - 1) * 16);
    };
    auto advance = [&](int c, f32x4_t& my_add, f32x4_t (&mine)[NDT]) {
        float* buf = state[(c - c0) & 1];
        *reinterpret_cast<f32x4_t*>(buf + l16 * kPitch + row) = cur;
        f32x4_t sum[2] = {my_add, f32x4_t{0.0f, 0.0f, 0.0f, 0.0f}}, now[NDT];
        if (kAhead == 2) {
#pragma unroll
            for (int k = 0; k < NDT; ++k) now[k] = mine[k];
            fetch(c + 2, my_add, mine);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (ok[r]) cs[c * pitch + from[r]] = cur[r];
        __syncthreads();
#pragma unroll
        for (int k = 0; k < NDT; ++k) {
            // (rows beyond dim are zero here, whatever stands in the matrix)
            const f32x4_t s4 = *reinterpret_cast<const f32x4_t*>(buf + l16 * kPitch + k * 16 + lq * 4);
#pragma unroll
            for (int r = 0; r < 4; ++r)
                sum[r & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(kAhead == 2 ? now[k][r] : mine[k][r], s4[r], sum[r & 1], 0, 0, 0);
        }
        if (kAhead == 1) fetch(c + 1, my_add, mine);
        cur = sum[0] + sum[1];
#pragma unroll
        for (int r = 0; r < 4; ++r) cur[r] = ok[r] ? cur[r] : 0.0f;
    };
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        ok[r] = row + r < dim && col < vdim;
        from[r] = ok[r] ? static_cast<int64_t>(row + r) * vdim + col : 0;
        cur[r] = ok[r] && !zero ? slot[from[r]] : 0.0f;
    }
#pragma unroll
    for (int i = 0; i < kAhead; ++i) fetch(c0 + i, add[i], m4[i]);
    for (int c = c0; c < c1; c += kAhead) {
#pragma unroll
        for (int i = 0; i < kAhead; ++i)
            if (c + i < c1) advance(c + i, add[i], m4[i]);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
        if (ok[r]) slot[from[r]] = cur[r];
}

// ---- decoding: one new token per sequence ----
// A thread holds VEC columns of up to ROWS rows of the state.
template <typename Elem, bool DELTA, int VEC, int ROWS>
__global__ __launch_bounds__(1024) void recur_step_kernel(RecurProblem p) {
    typedef typename Elem::storage S;
    typedef float vec_t __attribute__((ext_vector_type(VEC)));
    extern __shared__ __attribute__((aligned(16))) float lds[];
    __shared__ float red[2][16];
    const int dim = p.dim, vdim = p.vdim, threads = blockDim.x, waves = threads / kWave;
    const int cgs = vdim / VEC, groups = threads / cgs;
    float* lo = lds;                           // [groups][vdim]
    float* lv = lo + groups * vdim;            // [vdim]
    float* lqv = lv + vdim;                    // [dim] q
    float* lk = lqv + dim;                     // [dim] k
    const int tid = threadIdx.x, h = blockIdx.x, s = blockIdx.y, share = p.heads / p.kv_heads, g = h / share;
    const int grp = tid / cgs, c = (tid - grp * cgs) * VEC;
    const int pos = p.starts[s], slot = p.slots[s];
    float* st = p.states + (static_cast<int64_t>(slot) * p.heads + h) * dim * vdim;
    vec_t x[ROWS];
#pragma unroll
    for (int u = 0; u < ROWS; ++u) {
        const int d = grp + u * groups;
        if (grp < groups && d < dim && pos > 0) x[u] = *reinterpret_cast<const vec_t*>(st + d * vdim + c);
        else x[u] = static_cast<vec_t>(0.0f);
    }
    const f32x2_t rate = decay_and_beta<Elem>(p, s, h);
    const float decay = exp2_fast(rate[0]), beta = rate[1];

    const int64_t row = static_cast<int64_t>(s) * p.stride;
    const int channels = 2 * p.kv_heads * dim + p.heads * vdim;
    S* ring = static_cast<S*>(p.ring) + static_cast<int64_t>(slot) * p.taps * channels;
    float q_sum = 0.0f, k_sum = 0.0f;
    for (int i = tid; i < 2 * dim + vdim; i += threads) {
        const bool is_q = i < dim, is_k = !is_q && i < 2 * dim;
        const int at = is_q ? g * dim + i : is_k ? g * dim + i - dim : h * vdim + i - 2 * dim;
        const int channel = is_q ? at : is_k ? p.kv_heads * dim + at : 2 * p.kv_heads * dim + at;
        const S now = static_cast<const S*>(is_q ? p.q : is_k ? p.k : p.v)[row + at];
        const float* w = p.conv_w + static_cast<int64_t>(channel) * p.taps;
        float y = p.conv_b != nullptr ? p.conv_b[channel] : 0.0f;
        for (int back = min(p.taps - 1, pos); back > 0; --back)
            y = fmaf(w[p.taps - 1 - back], Elem::load(ring[static_cast<int64_t>((pos - back) % p.taps) * channels + channel]), y);
        y = silu(fmaf(w[p.taps - 1], Elem::load(now), y));
        // the projection's own row of the ring is read by nobody in this step
        if (!(is_q || is_k) || h % share == 0) ring[static_cast<int64_t>(pos % p.taps) * channels + channel] = now;
        if (is_q) {
            lqv[i] = y;
            q_sum = fmaf(y, y, q_sum);
        } else if (is_k) {
            lk[i - dim] = y;
            k_sum = fmaf(y, y, k_sum);
        } else {
            lv[i - 2 * dim] = Elem::load(Elem::store(y));
        }
    }
    float q_scale = p.q_scale, k_scale = 1.0f;
    if (p.unit_eps > 0.0f) {
        q_sum = wave_sum(q_sum);
        k_sum = wave_sum(k_sum);
        if ((tid & 63) == 0) {
            red[0][tid >> 6] = q_sum;
            red[1][tid >> 6] = k_sum;
        }
    }
    __syncthreads();
    if (p.unit_eps > 0.0f) {
        q_sum = k_sum = 0.0f;
        for (int w = 0; w < waves; ++w) {
            q_sum += red[0][w];
            k_sum += red[1][w];
        }
        q_scale /= sqrtf(q_sum + p.unit_eps);
        k_scale /= sqrtf(k_sum + p.unit_eps);
    }
    vec_t u_new = static_cast<vec_t>(0.0f);
    if (grp < groups) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) u_new[j] = lv[c + j];
    }
    if (DELTA) {
        vec_t sk = static_cast<vec_t>(0.0f);
#pragma unroll
        for (int u = 0; u < ROWS; ++u) {
            const int d = grp + u * groups;
            if (grp < groups && d < dim) {
                x[u] *= decay;
                sk += x[u] * (lk[d] * k_scale);
            }
        }
        if (grp < groups) *reinterpret_cast<vec_t*>(lo + grp * vdim + c) = sk;
        __syncthreads();
        if (grp < groups) {
            for (int w = 0; w < groups; ++w) u_new -= *reinterpret_cast<const vec_t*>(lo + w * vdim + c);
        }
        __syncthreads();
    }
    u_new *= beta;
    vec_t o = static_cast<vec_t>(0.0f);
#pragma unroll
    for (int u = 0; u < ROWS; ++u) {
        const int d = grp + u * groups;
        if (grp < groups && d < dim) {
            if (!DELTA) x[u] *= decay;
            x[u] += u_new * (lk[d] * k_scale);
            o += x[u] * (lqv[d] * q_scale);
            *reinterpret_cast<vec_t*>(st + d * vdim + c) = x[u];
        }
    }
    if (grp < groups) *reinterpret_cast<vec_t*>(lo + grp * vdim + c) = o;
    __syncthreads();
    float sum = 0.0f;
    for (int v = tid; v < vdim; v += threads) {
        float y = p.skip != nullptr ? p.skip[h] * lv[v] : 0.0f;
        for (int w = 0; w < groups; ++w) y += lo[w * vdim + v];
        lo[v] = y;                              // (column v is this thread's alone)
        sum = fmaf(y, y, sum);
    }
    float scale = 1.0f;
    if (DELTA) {
        sum = wave_sum(sum);
        if ((tid & 63) == 0) red[0][tid >> 6] = sum;      // (the unit vectors' sums were read before the last barriers)
        __syncthreads();
        sum = 0.0f;
        for (int w = 0; w < waves; ++w) sum += red[0][w];
        scale = 1.0f / sqrtf(sum / static_cast<float>(vdim) + p.eps);
    }
    for (int v = tid; v < vdim; v += threads) {
        float y = lo[v];
        if (DELTA) y *= scale * p.norm_w[v] * silu(Elem::load(static_cast<const S*>(p.gate)[row + h * vdim + v]));
        static_cast<S*>(p.out)[(static_cast<int64_t>(s) * p.heads + h) * vdim + v] = Elem::store(y);
    }
}

// ---- launches ----
template <typename Elem>
int launch_conv(const RecurProblem& p, hipStream_t s) {
    int head_lanes = 1;
    while (head_lanes * 4 < round_up(p.dim, 16)) head_lanes *= 2;
    const int units = static_cast<int>(2 * ceil_div(p.kv_heads, kWave / head_lanes) + ceil_div(p.heads * p.vdim, kConvPiece) + ceil_div(kBlock * p.heads, kWave));
    const dim3 grid(static_cast<unsigned>(p.n_chunks), static_cast<unsigned>(p.chunk_tokens / kBlock), static_cast<unsigned>(ceil_div(units, 4)));
    auto aligned = [](const void* ptr) { return reinterpret_cast<uintptr_t>(ptr) % (4 * sizeof(typename Elem::storage)) == 0; };
    const bool vec = p.dim % 4 == 0 && p.vdim % 4 == 0 && p.stride % 4 == 0 && aligned(p.q) && aligned(p.k) && aligned(p.v);
    if (p.taps > 4) launch((recur_conv_kernel<Elem, kMaxTaps, false>), grid, dim3(256), 0, s, p, head_lanes);
    else if (vec) launch((recur_conv_kernel<Elem, 4, true>), grid, dim3(256), 0, s, p, head_lanes);
    else launch((recur_conv_kernel<Elem, 4, false>), grid, dim3(256), 0, s, p, head_lanes);
    return launch_status();
}

template <typename Elem, int NDT, bool DELTA, bool OUTPUT, int THREADS>
int launch_chunks(const RecurProblem& p, int tiles, int waves, hipStream_t s) {
    const size_t lds = sizeof(float) * (static_cast<size_t>(OUTPUT ? 4 : 2) * kBlock * (NDT * 16 + 4) + 2 * waves * kBlock);
    const int rc = allow_lds(reinterpret_cast<const void*>(recur_chunk_kernel<Elem, NDT, DELTA, OUTPUT, THREADS>), lds);
    if (rc != 0) return rc;
    launch((recur_chunk_kernel<Elem, NDT, DELTA, OUTPUT, THREADS>),
           dim3(static_cast<unsigned>(p.n_chunks), static_cast<unsigned>(p.heads), static_cast<unsigned>(ceil_div(tiles, waves))),
           dim3(static_cast<unsigned>(waves * kWave)), lds, s, p);
    return launch_status();
}

template <typename Elem, int NDT, bool DELTA, bool OUTPUT>
int size_chunks(const RecurProblem& p, hipStream_t s) {
    const int v_tiles = static_cast<int>(ceil_div(p.vdim, 16));
    const int tiles = v_tiles + (DELTA && !OUTPUT ? static_cast<int>(ceil_div(p.dim, 16)) : 0);
    // (a head's norm needs all of its columns in one workgroup; at least four waves move the operands)
    if (DELTA && OUTPUT && tiles > 8) return launch_chunks<Elem, NDT, DELTA, OUTPUT, DELTA && OUTPUT ? 1024 : 512>(p, tiles, tiles, s);
    const int groups = static_cast<int>(ceil_div(tiles, 8));
    return launch_chunks<Elem, NDT, DELTA, OUTPUT, 512>(p, tiles, std::max(4, static_cast<int>(ceil_div(tiles, groups))), s);
}

template <typename Elem, bool DELTA, bool OUTPUT>
int dispatch_chunks(const RecurProblem& p, hipStream_t s) {
    if (p.dim <= 32) return size_chunks<Elem, 2, DELTA, OUTPUT>(p, s);
    if (p.dim <= 64) return size_chunks<Elem, 4, DELTA, OUTPUT>(p, s);
    if (p.dim <= 128) return size_chunks<Elem, 8, DELTA, OUTPUT>(p, s);
    return size_chunks<Elem, 16, DELTA, OUTPUT>(p, s);
}

template <bool DELTA>
int launch_scan(const RecurProblem& p, hipStream_t s) {
    const unsigned heads = static_cast<unsigned>(p.heads), seqs = static_cast<unsigned>(p.n_seqs);
    if (!DELTA) {
        launch(recur_scan_kernel, dim3(static_cast<unsigned>(ceil_div(p.dim * p.vdim, 256)), heads, seqs), dim3(256), 0, s, p);
        return launch_status();
    }
    const dim3 grid(heads, static_cast<unsigned>(ceil_div(p.vdim, 16)), seqs);
    if (p.dim <= 32) launch(recur_matrix_scan_kernel<2>, grid, dim3(2 * kWave), 0, s, p);
    else if (p.dim <= 64) launch(recur_matrix_scan_kernel<4>, grid, dim3(4 * kWave), 0, s, p);
    else if (p.dim <= 128) launch(recur_matrix_scan_kernel<8>, grid, dim3(8 * kWave), 0, s, p);
    else launch(recur_matrix_scan_kernel<16>, grid, dim3(16 * kWave), 0, s, p);
    return launch_status();
}

template <typename Elem, bool DELTA>
int prefill(const RecurProblem& p, hipStream_t s) {
    int rc = launch_conv<Elem>(p, s);
    if (rc != 0) return rc;
    int per_wave = kBlockHeads;
    while (p.heads / p.kv_heads % per_wave != 0) --per_wave;
    launch(recur_block_kernel<DELTA>, dim3(static_cast<unsigned>(p.n_chunks), static_cast<unsigned>(p.chunk_tokens / kBlock),
                                           static_cast<unsigned>(ceil_div(p.heads / per_wave, 4))), dim3(256), 0, s, p, per_wave);
    rc = launch_status();
    if (rc != 0) return rc;
    if (p.chunk_states != nullptr) {
        rc = dispatch_chunks<Elem, DELTA, false>(p, s);
        if (rc == 0) rc = launch_scan<DELTA>(p, s);
        if (rc != 0) return rc;
    }
    return dispatch_chunks<Elem, DELTA, true>(p, s);
}

template <typename Elem, bool DELTA, int VEC, int ROWS>
int launch_step(const RecurProblem& p, hipStream_t s) {
    const int cgs = p.vdim / VEC;
    int threads = 256;
    while (threads < 1024 && (threads / cgs == 0 || ceil_div(p.dim, threads / cgs) > ROWS)) threads *= 2;
    const size_t lds = sizeof(float) * (static_cast<size_t>(threads / cgs) * p.vdim + p.vdim + 2 * p.dim);
    launch((recur_step_kernel<Elem, DELTA, VEC, ROWS>), dim3(static_cast<unsigned>(p.heads), static_cast<unsigned>(p.n_seqs)),
           dim3(static_cast<unsigned>(threads)), lds, s, p);
    return launch_status();
}

template <typename Elem, bool DELTA>
int step(const RecurProblem& p, hipStream_t s) {
    return p.vdim % 4 == 0 ? launch_step<Elem, DELTA, 4, 16>(p, s) : launch_step<Elem, DELTA, 1, 64>(p, s);
}

}  // namespace

bool recur_supported(int heads, int kv_heads, int dim, int vdim, int taps) {
    return heads > 0 && heads <= 65535 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && dim <= 256 && vdim > 0 && vdim <= 256 &&
           taps > 0 && taps <= kMaxTaps;
}

int launch_recur_prefill(const RecurProblem& p, hipStream_t s) {
    if (p.dtype == EM_DTYPE_BF16) return p.beta_in ? prefill<BF16Elem, true>(p, s) : prefill<BF16Elem, false>(p, s);
    return p.beta_in ? prefill<F32Elem, true>(p, s) : prefill<F32Elem, false>(p, s);
}

int launch_recur_step(const RecurProblem& p, hipStream_t s) {
    if (p.dtype == EM_DTYPE_BF16) return p.beta_in ? step<BF16Elem, true>(p, s) : step<BF16Elem, false>(p, s);
    return p.beta_in ? step<F32Elem, true>(p, s) : step<F32Elem, false>(p, s);
}

}  // namespace em
