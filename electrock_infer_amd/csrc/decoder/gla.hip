// Gated linear attention: a recurrence with one decay per key channel,
//     S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,   alpha = sigmoid(z)^(1/tau),
// with a float32 state [dim, vdim] per head and sequence, an RMS norm of every head's output and a SiLU gate.
//
// Prompts.  A sequence's tokens are cut into chunks and a chunk into blocks of 16.  With bl_t the sum of log alpha from
// the block's first token to t (all values <= 0) and tot its last value, a block is
//     o_t   = (q_t exp(bl_t)) S  +  sum_{s <= t} [ sum_d q_td k_sd exp(bl_td - bl_sd) ] v_s
//     S    <- exp(tot) S + sum_s (k_s exp(tot - bl_s)) v_s^T
// which are float32 MFMAs: a wave keeps the state's 16 columns of one v tile in registers, in the layout in which an
// MFMA leaves its result; the same registers, as they are, are the second operand of the float32 16x16x4 MFMA.  One
// workgroup is one (chunk, head), one wave a v tile.  Everything that reaches the state is float32: the operands are
// products of the bf16 projections with float32 decays, and no exponent is positive except in the block's own 16 x 16
// scores, where exp(-bl_s) is used as a factor only while the whole block decays by less than 2^-kFactorLimit.  (The
// logarithms are kept to base 2.)
// With more than one chunk in a sequence the chunks run in parallel: a first pass leaves every chunk's own contribution
// to the state and its total decay, a scan over the chunks turns these into the states in front of them, and the
// output pass starts from there.
//
// Decoding.  One workgroup per (sequence, head) streams the state once: decay, update, read-out, norm and gate.
#include <type_traits>

#include "decoder.h"

namespace em {
namespace {

constexpr int kBlock = 16;
constexpr float kFactorLimit = 58.0f;  // log2
constexpr float kLog2e = 1.4426950408889634f;
constexpr int kPitchA = 20;   // floats between the rows of a 16 x 16 LDS matrix (16-byte reads of 4 columns)

__device__ __forceinline__ float exp2_fast(float x) { return __builtin_amdgcn_exp2f(x); }
// with the hardware's exponential and reciprocal, 1 ulp each
__device__ __forceinline__ float silu_fast(float g) { return g * __builtin_amdgcn_rcpf(1.0f + exp2_fast(-g * kLog2e)); }
__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.0f) - log1pf(expf(-fabsf(z))); }

// bl [T, C]: per channel (C = heads * dim) the running sum of log2 alpha inside every block of 16 tokens.
template <typename Elem>
__global__ __launch_bounds__(256) void gla_decay_kernel(const typename Elem::storage* __restrict__ a1, int64_t a1_stride,
                                                        const typename Elem::storage* __restrict__ a2, int rank, int a2_stride,
                                                        const float* __restrict__ bias, float inv_tau,
                                                        const int4* __restrict__ chunks, float* __restrict__ bl, int C) {
    extern __shared__ __attribute__((aligned(16))) float lds_a1[];  // [16][rank]
    const int4 ch = chunks[blockIdx.x];
    const int first = blockIdx.y * kBlock;
    if (first >= ch.z) return;
    const int n = min(kBlock, ch.z - first);
    const int64_t row0 = static_cast<int64_t>(ch.y) + first;
    for (int i = threadIdx.x; i < kBlock * rank; i += 256) {
        const int t = i / rank;
        lds_a1[i] = t < n ? Elem::load(a1[(row0 + t) * a1_stride + (i - t * rank)]) : 0.0f;
    }
    __syncthreads();
    const int c = blockIdx.z * 256 + threadIdx.x;
    if (c >= C) return;
    float z[kBlock];
    const float b = bias[c];
#pragma unroll
    for (int t = 0; t < kBlock; ++t) z[t] = b;
    const typename Elem::storage* w = a2 + static_cast<int64_t>(c) * a2_stride;
    if (rank % 4 == 0 && a2_stride % 4 == 0) {
        for (int j = 0; j < rank; j += 4) {
            typename Elem::storage ws[4];
            __builtin_memcpy(ws, __builtin_assume_aligned(w + j, sizeof(ws)), sizeof(ws));
#pragma unroll
            for (int t = 0; t < kBlock; ++t) {
                const f32x4_t a = *reinterpret_cast<const f32x4_t*>(lds_a1 + t * rank + j);
#pragma unroll
                for (int i = 0; i < 4; ++i) z[t] = fmaf(Elem::load(ws[i]), a[i], z[t]);
            }
        }
    } else {
        for (int j = 0; j < rank; ++j) {
            const float wj = Elem::load(w[j]);
#pragma unroll
            for (int t = 0; t < kBlock; ++t) z[t] = fmaf(wj, lds_a1[t * rank + j], z[t]);
        }
    }
    float sum = 0.0f;
#pragma unroll
    for (int t = 0; t < kBlock; ++t) {
        sum += log_sigmoid(z[t]) * (inv_tau * kLog2e);
        if (t < n) bl[(row0 + t) * C + c] = sum;
    }
}

// What the chunk kernels need to know; offsets and strides in elements.
struct GlaArgs {
    const void *q, *k, *v, *g;  // rows of `stride`, head h at h * dim (q, k) or h * vdim (v, g)
    int64_t stride;
    const float* bl;
    const float* norm_w;
    void* out;                  // [T, heads * vdim]
    const int4* chunks;         // {sequence, first row, tokens, unused}
    const int32_t* slots;       // state slot of every sequence
    const int32_t* starts;      // position of every sequence's first token in this step; 0: the state is zero
    float* states;              // [slots, heads, dim, vdim]
    float* chunk_states;        // [chunks, heads, dim, vdim]; null: one chunk per sequence, straight from / to the slots
    float* chunk_decay;         // [chunks, heads, dim] sum of log2 alpha
    int heads, dim, vdim;
    float q_scale, eps;
};

// What a thread of the chunk kernels loads for one block, ahead of its use: PAIRS pairs of neighbouring channels of q, k
// and bl, and four rows of this lane's v and g columns.
template <int PAIRS>
struct BlockRegs {
    uint32_t q[PAIRS], k[PAIRS];
    f32x2_t b[PAIRS], tot[PAIRS];
    uint16_t v[4], g[4];
};

// PAIRS > 0 (bf16, even dim, at most PAIRS * 2 * threads channel values per block, at most 512 threads): the next
// block's operands are in flight while this one is computed.  PAIRS == 0: any size, element by element.
template <typename Elem, int NDT, bool OUTPUT, int PAIRS>
__global__ __launch_bounds__(PAIRS > 0 ? 512 : 1024, PAIRS > 0 && NDT > 4 ? 2 : 4) void gla_chunk_kernel(GlaArgs p) {
    typedef typename Elem::storage S;
    constexpr int D = NDT * 16;
    constexpr int DP = D + 4;
    const int waves = blockDim.x / kWave;
    extern __shared__ float lds[];
    float* Qp = lds;                                  // [16][DP]  q exp(bl)
    float* Kn = Qp + kBlock * DP;                     // [16][DP]  k exp(-bl)
    float* Kt = Kn + kBlock * DP;                     // [D][20]   k exp(tot - bl), transposed
    float* Et = Kt + D * kPitchA;                     // [D]       exp(tot)
    float* Ap = Et + D;                               // [waves][16][20] partial scores
    float* Rs = Ap + waves * kBlock * kPitchA;        // [waves][16] partial row sums
    float* Bl = Rs + waves * kBlock;                  // [16][DP]  bl, for blocks with a large decay

    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int l16 = lane & 15, lq = lane >> 4;
    const int4 ch = p.chunks[blockIdx.x];
    const int h = blockIdx.y;
    const int dim = p.dim, vdim = p.vdim;
    const int vc = wave * 16 + l16;                   // this lane's state column
    const bool v_ok = vc < vdim;
    const S* qg = static_cast<const S*>(p.q) + static_cast<int64_t>(h) * dim;
    const S* kg = static_cast<const S*>(p.k) + static_cast<int64_t>(h) * dim;
    const S* vg = static_cast<const S*>(p.v) + static_cast<int64_t>(h) * vdim;
    const S* gg = static_cast<const S*>(p.g) + static_cast<int64_t>(h) * vdim;
    const int C = p.heads * dim;

    // state tile rows dt * 16 + lq * 4 + r, column vc
    f32x4_t st[NDT];
    const int64_t head_state = static_cast<int64_t>(dim) * vdim;
    float* slot = p.states + (static_cast<int64_t>(p.slots[ch.x]) * p.heads + h) * head_state;
    float* mine = p.chunk_states ? p.chunk_states + (static_cast<int64_t>(blockIdx.x) * p.heads + h) * head_state : slot;
    const bool from_zero = !OUTPUT || (p.chunk_states == nullptr && p.starts[ch.x] == 0);
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int d = dt * 16 + lq * 4 + r;
            st[dt][r] = (!from_zero && v_ok && d < dim) ? mine[static_cast<int64_t>(d) * vdim + vc] : 0.0f;
        }
    const float nw = (OUTPUT && v_ok) ? p.norm_w[vc] : 0.0f;
    const float inv_vdim = 1.0f / static_cast<float>(vdim);
    if (!OUTPUT)
        for (int d = tid; d < dim; d += blockDim.x) Bl[d] = 0.0f;  // here: the chunk's decay so far

    BlockRegs<PAIRS ? PAIRS : 1> regs;
    auto fetch = [&](int first) {
        const int n = min(kBlock, ch.z - first);
        const int64_t row0 = static_cast<int64_t>(ch.y) + first;
#pragma unroll
        for (int i = 0; i < PAIRS; ++i) {
            const int e = (tid + i * static_cast<int>(blockDim.x)) * 2, t = e / D, d = e - t * D;
            regs.q[i] = regs.k[i] = 0;
            regs.b[i] = regs.tot[i] = f32x2_t{0.0f, 0.0f};
            if (t < kBlock && d < dim) {
                regs.tot[i] = *reinterpret_cast<const f32x2_t*>(p.bl + (row0 + n - 1) * C + h * dim + d);
                regs.b[i] = regs.tot[i];
                if (t < n) {
                    regs.b[i] = *reinterpret_cast<const f32x2_t*>(p.bl + (row0 + t) * C + h * dim + d);
                    regs.k[i] = *reinterpret_cast<const uint32_t*>(kg + (row0 + t) * p.stride + d);
                    if (OUTPUT) regs.q[i] = *reinterpret_cast<const uint32_t*>(qg + (row0 + t) * p.stride + d);
                }
            }
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = lq * 4 + r;
            const bool ok = v_ok && t < n;
            regs.v[r] = ok ? static_cast<uint16_t>(vg[(row0 + t) * p.stride + vc]) : 0;
            if (OUTPUT) regs.g[r] = ok ? static_cast<uint16_t>(gg[(row0 + t) * p.stride + vc]) : 0;
        }
    };
    if (PAIRS > 0) fetch(0);

    for (int first = 0; first < ch.z; first += kBlock) {
        const int n = min(kBlock, ch.z - first);
        const int64_t row0 = static_cast<int64_t>(ch.y) + first;
        // ---- operands of the block ----
        bool factor_ok = true;
        auto place = [&](int t, int d, float q, float k, float b, float tot) {
            if (t == 0) Et[d] = exp2_fast(tot);
            Kt[d * kPitchA + t] = k * exp2_fast(tot - b);
            if (OUTPUT) {
                Qp[t * DP + d] = q * exp2_fast(b);
                Kn[t * DP + d] = k * exp2_fast(fminf(-b, kFactorLimit));
                factor_ok = factor_ok && tot > -kFactorLimit;
            }
        };
        float v[4], gate[4];
        if (PAIRS > 0) {
#pragma unroll
            for (int i = 0; i < PAIRS; ++i) {
                const int e = (tid + i * static_cast<int>(blockDim.x)) * 2, t = e / D, d = e - t * D;
                if (t < kBlock) {
                    place(t, d, bf16_lo(regs.q[i]) * p.q_scale, bf16_lo(regs.k[i]), regs.b[i][0], regs.tot[i][0]);
                    place(t, d + 1, bf16_hi(regs.q[i]) * p.q_scale, bf16_hi(regs.k[i]), regs.b[i][1], regs.tot[i][1]);
                }
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                v[r] = bf16_bits_to_f32(regs.v[r]);
                gate[r] = OUTPUT ? bf16_bits_to_f32(regs.g[r]) : 0.0f;
            }
            if (first + kBlock < ch.z) fetch(first + kBlock);
        } else {
            for (int i = tid; i < kBlock * D; i += blockDim.x) {
                const int t = i / D, d = i - t * D;
                float q = 0.0f, k = 0.0f, b = 0.0f, tot = 0.0f;
                if (d < dim) {
                    tot = p.bl[(row0 + n - 1) * C + h * dim + d];
                    b = tot;
                    if (t < n) {
                        b = p.bl[(row0 + t) * C + h * dim + d];
                        k = Elem::load(kg[(row0 + t) * p.stride + d]);
                        if (OUTPUT) q = Elem::load(qg[(row0 + t) * p.stride + d]) * p.q_scale;
                    }
                }
                place(t, d, q, k, b, tot);
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = lq * 4 + r;
                const bool ok = v_ok && t < n;
                v[r] = ok ? Elem::load(vg[(row0 + t) * p.stride + vc]) : 0.0f;
                gate[r] = OUTPUT && ok ? Elem::load(gg[(row0 + t) * p.stride + vc]) : 0.0f;
            }
        }
        if (OUTPUT) {
            factor_ok = __syncthreads_and(factor_ok);
            // ---- scores of the block, shared out over the waves by channel tile ----
            f32x4_t a = {0.0f, 0.0f, 0.0f, 0.0f};
            if (factor_ok) {
                for (int dt = wave; dt < NDT; dt += waves) {
                    const f32x4_t q4 = *reinterpret_cast<const f32x4_t*>(Qp + l16 * DP + dt * 16 + lq * 4);
                    const f32x4_t k4 = *reinterpret_cast<const f32x4_t*>(Kn + l16 * DP + dt * 16 + lq * 4);
#pragma unroll
                    for (int r = 0; r < 4; ++r) a = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[r], k4[r], a, 0, 0, 0);
                }
            } else {
                // pair by pair, with the difference of the exponents
                for (int i = tid; i < kBlock * D; i += blockDim.x) {
                    const int t = i / D, d = i - t * D;
                    Bl[t * DP + d] = (d < dim && t < n) ? p.bl[(row0 + t) * C + h * dim + d] : 0.0f;
                }
                __syncthreads();
#pragma unroll 1
                for (int r = 0; r < 4; ++r) {
                    const int t = lq * 4 + r, s = l16;
                    float sum = 0.0f;
                    if (s <= t && t < n) {
                        const S* qr = qg + (row0 + t) * p.stride;
                        const S* kr = kg + (row0 + s) * p.stride;
                        for (int d = wave; d < dim; d += waves)
                            sum += Elem::load(qr[d]) * p.q_scale * Elem::load(kr[d]) * exp2_fast(Bl[t * DP + d] - Bl[s * DP + d]);
                    }
                    a = f32x4_t{r == 0 ? sum : a[0], r == 1 ? sum : a[1], r == 2 ? sum : a[2], r == 3 ? sum : a[3]};
                }
            }
            // (waves beyond the channel tiles have nothing to add)
            if (wave < NDT || !factor_ok) {
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int t = lq * 4 + r;
                    Ap[(wave * kBlock + t) * kPitchA + l16] = l16 <= t ? a[r] : 0.0f;
                }
            }
        }
        __syncthreads();
        f32x4_t o = {0.0f, 0.0f, 0.0f, 0.0f};
        if (OUTPUT) {
            // ---- read-out of the state in front of the block, then the block's own part ----
#pragma unroll
            for (int dt = 0; dt < NDT; ++dt) {
                const f32x4_t q4 = *reinterpret_cast<const f32x4_t*>(Qp + l16 * DP + dt * 16 + lq * 4);
#pragma unroll
                for (int r = 0; r < 4; ++r) o = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[r], st[dt][r], o, 0, 0, 0);
            }
            f32x4_t a4 = {0.0f, 0.0f, 0.0f, 0.0f};
            const int parts = factor_ok ? min(waves, NDT) : waves;
            for (int w = 0; w < parts; ++w)
                a4 += *reinterpret_cast<const f32x4_t*>(Ap + (w * kBlock + l16) * kPitchA + lq * 4);
#pragma unroll
            for (int r = 0; r < 4; ++r) o = __builtin_amdgcn_mfma_f32_16x16x4f32(a4[r], v[r], o, 0, 0, 0);
        } else {
            for (int d = tid; d < dim; d += blockDim.x) Bl[d] += p.bl[(row0 + n - 1) * C + h * dim + d];
        }
        // ---- state behind the block ----
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) {
            const f32x4_t e4 = *reinterpret_cast<const f32x4_t*>(Et + dt * 16 + lq * 4);
            const f32x4_t k4 = *reinterpret_cast<const f32x4_t*>(Kt + (dt * 16 + l16) * kPitchA + lq * 4);
            st[dt] *= e4;
#pragma unroll
            for (int r = 0; r < 4; ++r) st[dt] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[r], v[r], st[dt], 0, 0, 0);
        }
        if (OUTPUT) {
            // ---- norm over the head's vdim outputs, gate ----
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                float ss = o[r] * o[r];
#pragma unroll
                for (int off = 8; off > 0; off >>= 1) ss += __shfl_xor(ss, off);
                if (l16 == 0) Rs[wave * kBlock + lq * 4 + r] = ss;
            }
        }
        __syncthreads();  // the block's LDS operands are no longer needed
        if (OUTPUT) {
            f32x4_t ss = {0.0f, 0.0f, 0.0f, 0.0f};
            for (int w = 0; w < waves; ++w) ss += *reinterpret_cast<const f32x4_t*>(Rs + w * kBlock + lq * 4);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = lq * 4 + r;
                if (v_ok && t < n) {
                    const float y = o[r] * __builtin_amdgcn_rsqf(ss[r] * inv_vdim + p.eps) * nw;
                    static_cast<S*>(p.out)[(row0 + t) * p.heads * vdim + h * vdim + vc] = Elem::store(y * silu_fast(gate[r]));
                }
            }
        }
    }
    if (!OUTPUT || p.chunk_states == nullptr) {
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int d = dt * 16 + lq * 4 + r;
                if (v_ok && d < dim) mine[static_cast<int64_t>(d) * vdim + vc] = st[dt][r];
            }
        if (!OUTPUT)
            for (int d = tid; d < dim; d += blockDim.x)
                p.chunk_decay[(static_cast<int64_t>(blockIdx.x) * p.heads + h) * dim + d] = Bl[d];
    }
}

// chunk_states: contribution of every chunk -> state in front of it; the state behind the last chunk goes to the slot.
__global__ __launch_bounds__(256) void gla_scan_kernel(GlaArgs p, const int32_t* __restrict__ seq_chunks) {
    constexpr int kAhead = 4;
    const int i = blockIdx.x * 256 + threadIdx.x;
    const int n = p.dim * p.vdim;
    if (i >= n) return;
    const int h = blockIdx.y, s = blockIdx.z, d = i / p.vdim;
    const int c0 = seq_chunks[s], c1 = seq_chunks[s + 1];
    const int64_t pitch = static_cast<int64_t>(p.heads) * n;
    float* slot = p.states + (static_cast<int64_t>(p.slots[s]) * p.heads + h) * n + i;
    float* cs = p.chunk_states + static_cast<int64_t>(h) * n + i;
    const float* cd = p.chunk_decay + static_cast<int64_t>(h) * p.dim + d;
    const int64_t dpitch = static_cast<int64_t>(p.heads) * p.dim;
    float state = p.starts[s] == 0 ? 0.0f : *slot;
    for (int c = c0; c < c1; c += kAhead) {
        float u[kAhead], e[kAhead];
#pragma unroll
        for (int j = 0; j < kAhead; ++j)
            if (c + j < c1) {
                u[j] = cs[(c + j) * pitch];
                e[j] = cd[(c + j) * dpitch];
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

// One new token per sequence.  VEC columns of the state per thread.
template <typename Elem, int VEC>
__global__ __launch_bounds__(256) void gla_step_kernel(GlaArgs p, const typename Elem::storage* __restrict__ a1,
                                                       const typename Elem::storage* __restrict__ a2, int rank,
                                                       int a2_stride, const float* __restrict__ bias, float inv_tau) {
    typedef typename Elem::storage S;
    typedef float vec_t __attribute__((ext_vector_type(VEC)));
    constexpr int kUnroll = 8;
    extern __shared__ float lds[];
    const int dim = p.dim, vdim = p.vdim;
    float* la = lds;              // [dim] alpha
    float* lq = la + dim;         // [dim]
    float* lk = lq + dim;         // [dim]
    float* lo = lk + dim;         // [groups][vdim]
    __shared__ float wave_sum[4];
    const int tid = threadIdx.x, h = blockIdx.x, s = blockIdx.y;
    const int64_t row = static_cast<int64_t>(s) * p.stride;
    const int C0 = h * dim;
    for (int d = tid; d < dim; d += 256) {
        const S* w = a2 + static_cast<int64_t>(C0 + d) * a2_stride;
        float z = bias[C0 + d];
        for (int j = 0; j < rank; ++j) z = fmaf(Elem::load(w[j]), Elem::load(a1[row + j]), z);
        la[d] = expf(log_sigmoid(z) * inv_tau);
        lq[d] = Elem::load(static_cast<const S*>(p.q)[row + C0 + d]) * p.q_scale;
        lk[d] = Elem::load(static_cast<const S*>(p.k)[row + C0 + d]);
    }
    __syncthreads();
    const int cgs = static_cast<int>(ceil_div(vdim, VEC));  // <= 256
    const int groups = 256 / cgs;
    const int grp = tid / cgs, c = (tid - grp * cgs) * VEC;
    const bool zero = p.starts[s] == 0;
    float* st = p.states + (static_cast<int64_t>(p.slots[s]) * p.heads + h) * dim * vdim;
    if (grp < groups) {
        float v[VEC], o[VEC];
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
            v[j] = Elem::load(static_cast<const S*>(p.v)[row + h * vdim + c + j]);
            o[j] = 0.0f;
        }
        for (int d0 = grp; d0 < dim; d0 += groups * kUnroll) {
            vec_t x[kUnroll];
#pragma unroll
            for (int u = 0; u < kUnroll; ++u) {
                const int d = d0 + u * groups;
                if (d < dim && !zero) x[u] = *reinterpret_cast<const vec_t*>(st + d * vdim + c);
                else x[u] = static_cast<vec_t>(0.0f);
            }
#pragma unroll
            for (int u = 0; u < kUnroll; ++u) {
                const int d = d0 + u * groups;
                if (d >= dim) continue;
                const float a = la[d], k = lk[d], q = lq[d];
#pragma unroll
                for (int j = 0; j < VEC; ++j) {
                    x[u][j] = fmaf(a, x[u][j], k * v[j]);
                    o[j] = fmaf(q, x[u][j], o[j]);
                }
                *reinterpret_cast<vec_t*>(st + d * vdim + c) = x[u];
            }
        }
#pragma unroll
        for (int j = 0; j < VEC; ++j) lo[grp * vdim + c + j] = o[j];
    }
    __syncthreads();
    float sum = 0.0f;
    for (int v = tid; v < vdim; v += 256) {
        float o = 0.0f;
        for (int g = 0; g < groups; ++g) o += lo[g * vdim + v];
        lo[v] = o;
        sum = fmaf(o, o, sum);
    }
#pragma unroll
    for (int off = kWave / 2; off > 0; off >>= 1) sum += __shfl_xor(sum, off);
    if ((tid & 63) == 0) wave_sum[tid >> 6] = sum;
    __syncthreads();
    const float rms = sqrtf((wave_sum[0] + wave_sum[1] + wave_sum[2] + wave_sum[3]) / static_cast<float>(vdim) + p.eps);
    for (int v = tid; v < vdim; v += 256) {
        const float g = Elem::load(static_cast<const S*>(p.g)[row + h * vdim + v]);
        static_cast<S*>(p.out)[(static_cast<int64_t>(s) * p.heads + h) * vdim + v] =
            Elem::store(lo[v] / rms * p.norm_w[v] * silu(g));
    }
}

size_t chunk_lds_bytes(int ndt, int waves) {
    const int D = ndt * 16, DP = D + 4;
    return sizeof(float) * (3 * kBlock * DP + D * kPitchA + D + waves * kBlock * kPitchA + waves * kBlock);
}

template <typename Elem, int NDT, bool OUTPUT, int PAIRS>
int launch_chunk_kernel(const GlaArgs& p, int n_chunks, hipStream_t s) {
    const int waves = static_cast<int>(ceil_div(p.vdim, 16));
    const dim3 grid(static_cast<unsigned>(n_chunks), static_cast<unsigned>(p.heads)), block(static_cast<unsigned>(waves * kWave));
    const size_t lds = chunk_lds_bytes(NDT, waves);
    const int rc = allow_lds(reinterpret_cast<const void*>(gla_chunk_kernel<Elem, NDT, OUTPUT, PAIRS>), lds);
    if (rc != 0) return rc;
    launch((gla_chunk_kernel<Elem, NDT, OUTPUT, PAIRS>), grid, block, lds, s, p);
    return launch_status();
}

template <typename Elem, int NDT>
int launch_chunks(const GlaArgs& p, int n_chunks, bool output, hipStream_t s) {
    const int threads = static_cast<int>(ceil_div(p.vdim, 16)) * kWave;
    const int pairs = static_cast<int>(ceil_div(kBlock * NDT * 16 / 2, threads));
    if (std::is_same<Elem, BF16Elem>::value && p.dim % 2 == 0 && pairs <= 2 && threads <= 512) {
        if (pairs == 1)
            return output ? launch_chunk_kernel<BF16Elem, NDT, true, 1>(p, n_chunks, s)
                          : launch_chunk_kernel<BF16Elem, NDT, false, 1>(p, n_chunks, s);
        return output ? launch_chunk_kernel<BF16Elem, NDT, true, 2>(p, n_chunks, s)
                      : launch_chunk_kernel<BF16Elem, NDT, false, 2>(p, n_chunks, s);
    }
    return output ? launch_chunk_kernel<Elem, NDT, true, 0>(p, n_chunks, s) : launch_chunk_kernel<Elem, NDT, false, 0>(p, n_chunks, s);
}

template <typename Elem>
int dispatch_chunks(const GlaArgs& p, int n_chunks, bool output, hipStream_t s) {
    if (p.dim <= 32) return launch_chunks<Elem, 2>(p, n_chunks, output, s);
    if (p.dim <= 64) return launch_chunks<Elem, 4>(p, n_chunks, output, s);
    if (p.dim <= 128) return launch_chunks<Elem, 8>(p, n_chunks, output, s);
    return launch_chunks<Elem, 16>(p, n_chunks, output, s);
}

GlaArgs make_args(const GlaProblem& g) {
    GlaArgs p;
    p.q = g.q; p.k = g.k; p.v = g.v; p.g = g.g;
    p.stride = g.stride;
    p.bl = g.bl;
    p.norm_w = g.norm_w;
    p.out = g.out;
    p.chunks = reinterpret_cast<const int4*>(g.chunks);
    p.slots = g.slots;
    p.starts = g.starts;
    p.states = g.states;
    p.chunk_states = g.chunk_states;
    p.chunk_decay = g.chunk_decay;
    p.heads = g.heads; p.dim = g.dim; p.vdim = g.vdim;
    p.q_scale = g.q_scale; p.eps = g.eps;
    return p;
}

}  // namespace

bool gla_supported(int heads, int dim, int vdim, int rank) {
    return heads > 0 && heads <= 65535 && dim > 0 && dim <= 256 && vdim > 0 && vdim <= 256 && rank > 0 && rank <= 512;
}

int launch_gla_prefill(const GlaProblem& g, const int32_t* seq_chunks, int n_chunks, int n_seqs, int chunk_tokens,
                       hipStream_t s) {
    const GlaArgs p = make_args(g);
    const int C = g.heads * g.dim;
    const dim3 dgrid(static_cast<unsigned>(n_chunks), static_cast<unsigned>(chunk_tokens / kBlock),
                     static_cast<unsigned>(ceil_div(C, 256)));
    const size_t dlds = sizeof(float) * kBlock * g.rank;
    if (g.dtype == EM_DTYPE_BF16)
        launch((gla_decay_kernel<BF16Elem>), dgrid, dim3(256), dlds, s, static_cast<const uint16_t*>(g.a1), g.stride,
               static_cast<const uint16_t*>(g.a2), g.rank, g.a2_stride, g.bias, 1.0f / g.tau, p.chunks, g.bl, C);
    else
        launch((gla_decay_kernel<F32Elem>), dgrid, dim3(256), dlds, s, static_cast<const float*>(g.a1), g.stride,
               static_cast<const float*>(g.a2), g.rank, g.a2_stride, g.bias, 1.0f / g.tau, p.chunks, g.bl, C);
    int rc = launch_status();
    if (rc != 0) return rc;
    if (g.chunk_states != nullptr) {
        rc = g.dtype == EM_DTYPE_BF16 ? dispatch_chunks<BF16Elem>(p, n_chunks, false, s)
                                      : dispatch_chunks<F32Elem>(p, n_chunks, false, s);
        if (rc != 0) return rc;
        launch(gla_scan_kernel, dim3(static_cast<unsigned>(ceil_div(g.dim * g.vdim, 256)), static_cast<unsigned>(g.heads),
                                     static_cast<unsigned>(n_seqs)), dim3(256), 0, s, p, seq_chunks);
        rc = launch_status();
        if (rc != 0) return rc;
    }
    return g.dtype == EM_DTYPE_BF16 ? dispatch_chunks<BF16Elem>(p, n_chunks, true, s)
                                    : dispatch_chunks<F32Elem>(p, n_chunks, true, s);
}

int launch_gla_step(const GlaProblem& g, int n_seqs, hipStream_t s) {
    const GlaArgs p = make_args(g);
    const dim3 grid(static_cast<unsigned>(g.heads), static_cast<unsigned>(n_seqs));
    const int vec = g.vdim % 4 == 0 ? 4 : 1;
    const int groups = 256 / static_cast<int>(ceil_div(g.vdim, vec));
    const size_t lds = sizeof(float) * (3 * g.dim + groups * g.vdim);
#define EM_STEP(E, V)                                                                                                \
    launch((gla_step_kernel<E, V>), grid, dim3(256), lds, s, p, static_cast<const typename E::storage*>(g.a1),       \
           static_cast<const typename E::storage*>(g.a2), g.rank, g.a2_stride, g.bias, 1.0f / g.tau)
    if (g.dtype == EM_DTYPE_BF16) {
        if (vec == 4) EM_STEP(BF16Elem, 4);
        else EM_STEP(BF16Elem, 1);
    } else {
        if (vec == 4) EM_STEP(F32Elem, 4);
        else EM_STEP(F32Elem, 1);
    }
#undef EM_STEP
    return launch_status();
}

}  // namespace em
