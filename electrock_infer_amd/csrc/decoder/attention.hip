// Softmax attention over a paged cache of keys and values, grouped heads: query head h uses key/value head
// h / (heads / kv_heads).  Optional: an RMS norm of every query and key head, a rotation of neighbouring pairs, a soft cap
// on the scores, a sliding window, and values mixed with those of an earlier layer.
//
// The cache holds, per token, the kv_heads keys (each padded with zeros to eight elements) and behind them the values.
// Both attention kernels compute S^T = K Q^T per tile of keys: a lane then holds, for one query, keys (lane / 16) * 4 +
// 0..3 of every 16, and since a sum over keys may run in any order as long as both operands agree, these registers are
// the second operand of O^T = V^T P^T as they are.  V^T comes out of LDS, where the values lie key by key, with
// transposing reads.
//
// paged_kernel: any portion, both types; a wave takes tiles of 32 keys for 16 (token, head) rows that share a key/value
// head, on its own, and the workgroup's four waves add up at the end.  prompt_kernel: long portions, bf16; 128 queries of
// a head per workgroup, 32 per wave, tiles of 64 keys shared by the four waves.
#include "decoder.h"
#include "mma.h"

namespace em {
namespace {

constexpr float kLog2e = 1.4426950408889634f;
constexpr float kFixedCap = 40.0f;    // up to here exp(-2 cap) is a normal float32: the cap itself can stand for the maximum

__device__ __forceinline__ float exp2_fast(float x) { return __builtin_amdgcn_exp2f(x); }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int off = kWave / 2; off > 0; off >>= 1) v += __shfl_xor(v, off);
    return v;
}

// ---- norms, rotation, mixing, cache write ----
// One workgroup, or for few tokens several, per token; a wave per head.  PAIR: heads begin at a multiple of two elements.
template <typename Elem, bool PAIR>
__global__ __launch_bounds__(256) void attn_prepare_kernel(AttnProblem p) {
    typedef typename Elem::storage S;
    constexpr int kPairs = 2;        // per lane: heads of up to 256 elements
    extern __shared__ float cs[];    // [rot / 2] cosines, [rot / 2] sines
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x, lane = tid & 63, half = p.rot / 2, dim = p.dim;
    const float pos = static_cast<float>(p.positions[t]);
    for (int i = tid; i < half; i += 256) {
        float sn, c;
        sincosf(pos * p.inv_freq[i], &sn, &c);
        cs[i] = c;
        cs[half + i] = sn;
    }
    __syncthreads();
    const int dp = attn_pitch(dim), vp = attn_pitch(p.vdim), row = attn_row_elems(p.kv_heads, dim, p.vdim);
    S* cached = static_cast<S*>(p.cache) + static_cast<int64_t>(p.cache_rows[t]) * row;
    for (int u = blockIdx.y * 4 + (tid >> 6); u < p.heads + p.kv_heads; u += 4 * gridDim.y) {
        const bool is_q = u < p.heads;
        const int h = is_q ? u : u - p.heads;
        const S* src = static_cast<const S*>(is_q ? p.q : p.k) + t * p.stride + h * dim;
        const float* w = is_q ? p.q_norm : p.k_norm;
        S* dst = is_q ? static_cast<S*>(p.q_out) + (t * p.heads + h) * dp : cached + h * dp;
        float a[kPairs], b[kPairs], ss = 0.0f;
#pragma unroll
        for (int i = 0; i < kPairs; ++i) {
            const int c = (lane + i * kWave) * 2;
            if (PAIR) {
                S two[2] = {0, 0};
                if (c < dim) __builtin_memcpy(two, __builtin_assume_aligned(src + c, sizeof(two)), sizeof(two));
                a[i] = Elem::load(two[0]);
                b[i] = Elem::load(two[1]);
            } else {
                a[i] = c < dim ? Elem::load(src[c]) : 0.0f;
                b[i] = c + 1 < dim ? Elem::load(src[c + 1]) : 0.0f;
            }
            ss = fmaf(a[i], a[i], fmaf(b[i], b[i], ss));
        }
        if (w != nullptr) {
            const float rstd = 1.0f / sqrtf(wave_sum(ss) / static_cast<float>(dim) + p.eps);
#pragma unroll
            for (int i = 0; i < kPairs; ++i) {
                const int c = (lane + i * kWave) * 2;
                if (c < dim) a[i] *= rstd * w[c];
                if (c + 1 < dim) b[i] *= rstd * w[c + 1];
            }
        }
#pragma unroll
        for (int i = 0; i < kPairs; ++i) {
            const int pair = lane + i * kWave;
            if (pair * 2 >= dp) continue;
            float x = a[i], y = b[i];
            if (pair < half) {
                x = a[i] * cs[pair] - b[i] * cs[half + pair];
                y = b[i] * cs[pair] + a[i] * cs[half + pair];
            }
            S two[2] = {Elem::store(x), Elem::store(y)};
            __builtin_memcpy(__builtin_assume_aligned(dst + pair * 2, sizeof(two)), two, sizeof(two));
        }
    }
    const float lambda = p.mix != nullptr ? *p.mix : 0.0f;
    S* values = cached + p.kv_heads * dp;
    for (int i = blockIdx.y * 256 + tid; i < p.kv_heads * vp; i += 256 * gridDim.y) {
        const int g = i / vp, c = i - g * vp;
        float v = 0.0f;
        if (c < p.vdim) {
            v = Elem::load(static_cast<const S*>(p.v)[t * p.stride + g * p.vdim + c]);
            if (p.mix != nullptr)
                v = (1.0f - lambda) * v + lambda * Elem::load(static_cast<const S*>(p.v_first)[t * p.v_first_stride + g * p.vdim + c]);
        }
        values[i] = Elem::store(v);
    }
}

// Columns col0 + l16 of two groups of four rows of an LDS matrix, as one operand fragment.
template <typename Elem>
__device__ __forceinline__ typename Mma<Elem>::frag load_columns(const typename Elem::storage* m, int pitch, int row_lo, int row_hi,
                                                                 int col0, int l16);
template <>
__device__ __forceinline__ f32x8_t load_columns<F32Elem>(const float* m, int pitch, int row_lo, int row_hi, int col0, int l16) {
    f32x8_t f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        f[i] = m[(row_lo + i) * pitch + col0 + l16];
        f[i + 4] = m[(row_hi + i) * pitch + col0 + l16];
    }
    return f;
}
template <>
__device__ __forceinline__ bf16x8_t load_columns<BF16Elem>(const uint16_t* m, int pitch, int row_lo, int row_hi, int col0, int l16) {
    // ds_read_b64_tr_b16: the 16 lanes of a group name the four-element pieces of a 4 x 16 block, row by row, and lane i
    // receives column i of it
    typedef short s16x4_t __attribute__((ext_vector_type(4)));
    typedef __attribute__((address_space(3))) s16x4_t* lds_ptr;
    const uint16_t* a = m + (l16 >> 2) * pitch + col0 + (l16 & 3) * 4;
    const s16x4_t lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)(a + row_lo * pitch));
    const s16x4_t hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)(a + row_hi * pitch));
    bf16x8_t f;
    __builtin_memcpy(&f, &lo, 8);
    __builtin_memcpy(reinterpret_cast<char*>(&f) + 8, &hi, 8);
    return f;
}

template <typename Elem> struct Precise;
template <> struct Precise<F32Elem> {
    static __device__ __forceinline__ float exp(float x) { return expf(x); }
    static __device__ __forceinline__ float cap(float s, float cap) { return cap * tanhf(s / cap); }
};
template <> struct Precise<BF16Elem> {    // the hardware's exponential and reciprocal, 1 ulp each
    static __device__ __forceinline__ float exp(float x) { return exp2_fast(x * kLog2e); }
    static __device__ __forceinline__ float cap(float s, float cap) {
        return cap - 2.0f * cap * __builtin_amdgcn_rcpf(exp2_fast(s / cap * (2.0f * kLog2e)) + 1.0f);
    }
};

// ---- any portion ----
constexpr int kKeys = 32;
template <typename Elem> __host__ __device__ constexpr int value_pitch(int dvt) { return dvt * 16 + 16 / static_cast<int>(sizeof(typename Elem::storage)); }
template <typename Elem> __host__ __device__ constexpr int paged_lds(int dvt) {   // values of a wave's tile; later the waves' results
    return 4 * kKeys * value_pitch<Elem>(dvt) * static_cast<int>(sizeof(typename Elem::storage)) > 4 * 16 * (dvt * 16 + 4) * 4
               ? 4 * kKeys * value_pitch<Elem>(dvt) * static_cast<int>(sizeof(typename Elem::storage)) : 4 * 16 * (dvt * 16 + 4) * 4;
}

// DKT: 32-element steps of dim; DVT: 16-element tiles of vdim
template <typename Elem, int DKT, int DVT>
__global__ __launch_bounds__(256, sizeof(typename Elem::storage) == 2 ? 2 : 1) void attn_paged_kernel(AttnProblem p, int splits,
                                                                                                    float* __restrict__ part_o,
                                                                                                    float* __restrict__ part_ml) {
    typedef typename Elem::storage S;
    typedef Mma<Elem> M;
    constexpr int LPV = value_pitch<Elem>(DVT), kPieces = kKeys * DVT * 2 / kWave, LPO = DVT * 16 + 4;
    extern __shared__ __attribute__((aligned(16))) uint8_t lds_raw[];
    __shared__ float wave_m[4][16], wave_l[4][16];
    const int share = p.heads / p.kv_heads;
    const int seq = blockIdx.y / p.kv_heads, g = blockIdx.y - seq * p.kv_heads, split = blockIdx.z;
    const int q0 = p.q_begin[seq], rows = (p.q_begin[seq + 1] - q0) * share, r0 = blockIdx.x * 16;
    if (r0 >= rows) return;
    const int start = p.starts[seq];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lq = lane >> 4;
    const int first_pos = start + r0 / share, last_pos = start + min(r0 + 15, rows - 1) / share;
    const int lowest = p.window > 0 ? max(0, first_pos - p.window + 1) : 0;
    const int tile_lo = lowest / kKeys, n_tiles = last_pos / kKeys + 1 - tile_lo;
    const int per_split = (n_tiles + splits - 1) / splits;
    const int tile0 = tile_lo + split * per_split, tile1 = tile_lo + min((split + 1) * per_split, n_tiles);
    const int dp = attn_pitch(p.dim), vp = attn_pitch(p.vdim), row_elems = attn_row_elems(p.kv_heads, p.dim, p.vdim);

    // this lane's query: row l16
    const int mine = min(r0 + l16, rows - 1), my_t = mine / share, my_h = g * share + mine - my_t * share;
    const int pos = start + my_t, low = p.window > 0 ? pos - p.window + 1 : 0;
    typename M::frag fq[DKT];
    {
        const S* q = static_cast<const S*>(p.q_out) + ((static_cast<int64_t>(q0) + my_t) * p.heads + my_h) * dp;
#pragma unroll
        for (int k = 0; k < DKT; ++k) fq[k] = k * 32 + lq * 8 < dp ? M::load(q + k * 32 + lq * 8) : M::zero();
    }
    f32x4_t o[DVT];
#pragma unroll
    for (int d = 0; d < DVT; ++d) o[d] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
    float m = -INFINITY, l = 0.0f;       // l: this lane's share
    S* Vs = reinterpret_cast<S*>(lds_raw) + wave * kKeys * LPV;
    const int32_t* table = p.tables + static_cast<int64_t>(seq) * p.table_width;
    const S* keys = static_cast<const S*>(p.cache) + g * dp;
    const S* values = static_cast<const S*>(p.cache) + p.kv_heads * dp + g * vp;
    const int pieces = vp / 8;
    auto row_of = [&](int tile) {
        const int key = tile * kKeys + (lane & 31);
        return key <= last_pos && tile < tile1 ? table[key / p.block_size] * p.block_size + key % p.block_size : -1;
    };
    int next_row = row_of(tile0 + wave);
    for (int tile = tile0 + wave; tile < tile1; tile += 4) {
        const int row = next_row;
        next_row = row_of(tile + 4);
        typename M::frag fv[kPieces];
#pragma unroll
        for (int i = 0; i < kPieces; ++i) {
            const int e = lane + i * kWave, key = e / pieces, c = (e - key * pieces) * 8;
            const int r = __shfl(row, key & 31);
            fv[i] = key < kKeys && r >= 0 ? M::load(values + static_cast<int64_t>(r) * row_elems + c) : M::zero();
        }
        f32x4_t s[2];
#pragma unroll
        for (int n = 0; n < 2; ++n) {
            s[n] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
            const int r = __shfl(row, n * 16 + l16);
            const S* kr = keys + static_cast<int64_t>(max(r, 0)) * row_elems;
#pragma unroll
            for (int k = 0; k < DKT; ++k) {
                const int c = k * 32 + lq * 8;
                s[n] = M::mac(c < dp && r >= 0 ? M::load(kr + c) : M::zero(), fq[k], s[n]);
            }
        }
#pragma unroll
        for (int i = 0; i < kPieces; ++i) {
            const int e = lane + i * kWave, key = e / pieces, c = (e - key * pieces) * 8;
            if (key < kKeys) store_frag<Elem>(Vs + key * LPV + c, fv[i]);
        }
        float mx = -INFINITY;
#pragma unroll
        for (int n = 0; n < 2; ++n)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int key = tile * kKeys + n * 16 + lq * 4 + r;
                float v = s[n][r] * p.scale;
                if (p.softcap > 0.0f) v = Precise<Elem>::cap(v, p.softcap);
                s[n][r] = key <= pos && key >= low ? v : -INFINITY;
                mx = fmaxf(mx, s[n][r]);
            }
        mx = fmaxf(mx, __shfl_xor(mx, 16));
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        const float mn = fmaxf(m, mx), base = mn == -INFINITY ? 0.0f : mn;
        const float alpha = Precise<Elem>::exp(m - base);
        m = mn;
        typename M::frag fp;
        float sum = 0.0f;
#pragma unroll
        for (int n = 0; n < 2; ++n)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const float e = Precise<Elem>::exp(s[n][r] - base);
                sum += e;
                M::set(fp, n * 4 + r, Elem::store(e));
            }
        l = l * alpha + sum;
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");       // this wave's values are its own
#pragma unroll
        for (int d = 0; d < DVT; ++d) {
            if (d * 16 < vp) {
                o[d] *= alpha;
                o[d] = M::mac(load_columns<Elem>(Vs, LPV, lq * 4, 16 + lq * 4, d * 16, l16), fp, o[d]);
            }
        }
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    }
    l += __shfl_xor(l, 16);
    l += __shfl_xor(l, 32);
    if (lq == 0) {
        wave_m[wave][l16] = m;
        wave_l[wave][l16] = l;
    }
    __syncthreads();
    float* Os = reinterpret_cast<float*>(lds_raw);                   // [4][16][LPO]
#pragma unroll
    for (int d = 0; d < DVT; ++d)
        *reinterpret_cast<f32x4_t*>(Os + (wave * 16 + l16) * LPO + d * 16 + lq * 4) = o[d];
    __syncthreads();
    for (int i = tid; i < 16 * DVT * 16; i += 256) {
        const int rr = i / (DVT * 16), c = i - rr * (DVT * 16);
        if (r0 + rr >= rows || c >= p.vdim) continue;
        const float top = fmaxf(fmaxf(wave_m[0][rr], wave_m[1][rr]), fmaxf(wave_m[2][rr], wave_m[3][rr]));
        const float base = top == -INFINITY ? 0.0f : top;
        float sum = 0.0f, v = 0.0f;
#pragma unroll
        for (int w = 0; w < 4; ++w) {
            const float weight = Precise<Elem>::exp(wave_m[w][rr] - base);
            sum = fmaf(wave_l[w][rr], weight, sum);
            v = fmaf(Os[(w * 16 + rr) * LPO + c], weight, v);
        }
        const int t = (r0 + rr) / share, h = g * share + r0 + rr - t * share;
        const int64_t row = (static_cast<int64_t>(q0) + t) * p.heads + h;
        if (splits == 1) {
            static_cast<S*>(p.out)[row * p.vdim + c] = Elem::store(v / sum);
        } else {
            part_o[(row * splits + split) * p.vdim + c] = v;
            if (c == 0) {
                part_ml[(row * splits + split) * 2] = top;
                part_ml[(row * splits + split) * 2 + 1] = sum;
            }
        }
    }
}

template <typename Elem>
__global__ __launch_bounds__(64) void attn_combine_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml, int splits,
                                                          int vdim, typename Elem::storage* __restrict__ out) {
    constexpr int kAhead = 8;
    __shared__ float weight[kAttnMaxSplits];
    const int64_t row = blockIdx.x;
    const float* ml = part_ml + row * splits * 2;
    const int lane = threadIdx.x;                                    // splits <= 64
    const float mine = lane < splits ? ml[2 * lane] : -INFINITY;
    float top = mine;
#pragma unroll
    for (int off = kWave / 2; off > 0; off >>= 1) top = fmaxf(top, __shfl_xor(top, off));
    const float e = lane < splits ? expf(mine - top) : 0.0f;
    const float den = wave_sum(lane < splits ? ml[2 * lane + 1] * e : 0.0f);
    weight[lane] = e / den;
    __syncthreads();
    for (int c = lane; c < vdim; c += kWave) {
        const float* src = part_o + row * splits * vdim + c;
        float v = 0.0f;
        for (int s0 = 0; s0 < splits; s0 += kAhead) {
            float x[kAhead];
#pragma unroll
            for (int j = 0; j < kAhead; ++j) x[j] = s0 + j < splits ? src[static_cast<int64_t>(s0 + j) * vdim] : 0.0f;
#pragma unroll
            for (int j = 0; j < kAhead; ++j)
                if (s0 + j < splits) v = fmaf(x[j], weight[s0 + j], v);
        }
        out[row * vdim + c] = Elem::store(v);
    }
}

// ---- long portions ----
constexpr int kTileKeys = 64;
constexpr int kRowsPerWave = 32;
constexpr int kRows = 4 * kRowsPerWave;

template <int DKT, int DVT>
__global__ __launch_bounds__(256, 2) void attn_prompt_kernel(AttnProblem p) {
    typedef Mma<BF16Elem> M;
    constexpr int LPK = DKT * 32 + 8, LPV = DVT * 16 + 8;
    constexpr int kFetchK = kTileKeys * DKT * 4 / 256, kFetchV = kTileKeys * DVT * 2 / 256;
    __shared__ __attribute__((aligned(16))) uint16_t Ks[kTileKeys * LPK];
    __shared__ __attribute__((aligned(16))) uint16_t Vs[kTileKeys * LPV];
    __shared__ int Kr[2][kTileKeys];                                 // cache row of every key of a tile, -1: no key
    const int h = blockIdx.x, seq = blockIdx.z, g = h / (p.heads / p.kv_heads);
    const int row0 = p.q_begin[seq], nq = p.q_begin[seq + 1] - row0;
    const int t0 = (static_cast<int>(gridDim.y) - 1 - static_cast<int>(blockIdx.y)) * kRows;  // long rows start first
    if (t0 >= nq) return;
    const int start = p.starts[seq];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lq = lane >> 4;
    const int dp = attn_pitch(p.dim), vp = attn_pitch(p.vdim), row_elems = attn_row_elems(p.kv_heads, p.dim, p.vdim);
    const int last_pos = start + min(t0 + kRows, nq) - 1;
    const int window = p.window > 0 ? p.window : last_pos + 1;
    const int tile0 = max(0, start + t0 - window + 1) / kTileKeys, tile1 = last_pos / kTileKeys + 1;
    const int first_pos = start + t0 + wave * kRowsPerWave;          // of this wave's first query

    typename M::frag fq[2][DKT];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
        const int t = min(t0 + wave * kRowsPerWave + j * 16 + l16, nq - 1);
        const uint16_t* q = static_cast<const uint16_t*>(p.q_out) + ((row0 + static_cast<int64_t>(t)) * p.heads + h) * dp;
#pragma unroll
        for (int k = 0; k < DKT; ++k) {
            const int c = k * 32 + lq * 8;
            fq[j][k] = c < dp ? M::load(q + c) : M::zero();
        }
    }
    const int32_t* table = p.tables + static_cast<int64_t>(seq) * p.table_width;
    const uint16_t* keys = static_cast<const uint16_t*>(p.cache) + g * dp;
    const uint16_t* values = static_cast<const uint16_t*>(p.cache) + p.kv_heads * dp + g * vp;
    auto find_rows = [&](int tile) {
        if (tid < kTileKeys && tile < tile1) {
            const int key = tile * kTileKeys + tid;
            Kr[tile & 1][tid] = key <= last_pos ? table[key / p.block_size] * p.block_size + key % p.block_size : -1;
        }
    };
    typename M::frag rk[kFetchK], rv[kFetchV];
    auto fetch = [&](int tile) {
#pragma unroll
        for (int i = 0; i < kFetchK; ++i) {
            const int e = tid + i * 256, c = (e % (DKT * 4)) * 8, row = Kr[tile & 1][e / (DKT * 4)];
            rk[i] = c < dp && row >= 0 ? M::load(keys + static_cast<int64_t>(row) * row_elems + c) : M::zero();
        }
#pragma unroll
        for (int i = 0; i < kFetchV; ++i) {
            const int e = tid + i * 256, c = (e % (DVT * 2)) * 8, row = Kr[tile & 1][e / (DVT * 2)];
            rv[i] = c < vp && row >= 0 ? M::load(values + static_cast<int64_t>(row) * row_elems + c) : M::zero();
        }
    };
    f32x4_t o[DVT][2];
#pragma unroll
    for (int d = 0; d < DVT; ++d) o[d][0] = o[d][1] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
    const bool capped = p.softcap > 0.0f, fixed = capped && p.softcap <= kFixedCap;
    const float c2 = p.scale * kLog2e, cap2 = p.softcap * kLog2e, in_cap = capped ? 2.0f * kLog2e * p.scale / p.softcap : 0.0f;
    // running maxima in units of log2 (the cap is one that never has to be raised); l: this lane's share
    float m[2], l[2] = {0.0f, 0.0f};
    m[0] = m[1] = fixed ? cap2 : -INFINITY;

    find_rows(tile0);
    find_rows(tile0 + 1);
    __syncthreads();
    fetch(tile0);
    for (int tile = tile0; tile < tile1; ++tile) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < kFetchK; ++i) {
            const int e = tid + i * 256;
            store_frag<BF16Elem>(Ks + (e / (DKT * 4)) * LPK + (e % (DKT * 4)) * 8, rk[i]);
        }
#pragma unroll
        for (int i = 0; i < kFetchV; ++i) {
            const int e = tid + i * 256;
            store_frag<BF16Elem>(Vs + (e / (DVT * 2)) * LPV + (e % (DVT * 2)) * 8, rv[i]);
        }
        if (tile + 1 < tile1) fetch(tile + 1);
        __syncthreads();
        find_rows(tile + 2);     // into the half that this tile's rows leave; read behind the next barriers
        const int k0 = tile * kTileKeys;
        // no key of this tile for this wave's queries
        if (k0 > first_pos + kRowsPerWave - 1 || k0 + kTileKeys - 1 < first_pos - window + 1) continue;

        f32x4_t s[4][2];
#pragma unroll
        for (int n = 0; n < 4; ++n) s[n][0] = s[n][1] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int k = 0; k < DKT; ++k)
#pragma unroll
            for (int n = 0; n < 4; ++n) {
                const typename M::frag fk = M::load(Ks + (n * 16 + l16) * LPK + k * 32 + lq * 8);
                s[n][0] = M::mac(fk, fq[0][k], s[n][0]);
                s[n][1] = M::mac(fk, fq[1][k], s[n][1]);
            }
        // scores in units of log2
        if (capped) {
#pragma unroll
            for (int n = 0; n < 4; ++n)
#pragma unroll
                for (int j = 0; j < 2; ++j)
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        s[n][j][r] = fmaf(-2.0f * cap2, __builtin_amdgcn_rcpf(exp2_fast(s[n][j][r] * in_cap) + 1.0f), cap2);
        } else {
#pragma unroll
            for (int n = 0; n < 4; ++n) {
                s[n][0] *= c2;
                s[n][1] *= c2;
            }
        }
        if (k0 + kTileKeys - 1 > first_pos || k0 < first_pos + kRowsPerWave - window) {
#pragma unroll
            for (int n = 0; n < 4; ++n)
#pragma unroll
                for (int j = 0; j < 2; ++j)
#pragma unroll
                    for (int r = 0; r < 4; ++r) {
                        const int gap = first_pos + j * 16 + l16 - (k0 + n * 16 + lq * 4 + r);
                        if (gap < 0 || gap >= window) s[n][j][r] = -INFINITY;
                    }
        }
        typename M::frag fp[2][2];   // [32-key step][query tile]
        float alpha[2] = {1.0f, 1.0f};
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            float base = m[j];
            if (!fixed) {
                float mx = -INFINITY;
#pragma unroll
                for (int n = 0; n < 4; ++n)
#pragma unroll
                    for (int r = 0; r < 4; ++r) mx = fmaxf(mx, s[n][j][r]);
                mx = fmaxf(mx, __shfl_xor(mx, 16));
                mx = fmaxf(mx, __shfl_xor(mx, 32));
                const float mn = fmaxf(m[j], mx);
                base = mn == -INFINITY ? 0.0f : mn;
                alpha[j] = exp2_fast(m[j] - base);
                m[j] = mn;
            }
            float sum = 0.0f;
#pragma unroll
            for (int n = 0; n < 4; ++n)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float e = exp2_fast(s[n][j][r] - base);
                    sum += e;
                    fp[n >> 1][j][(n & 1) * 4 + r] = static_cast<__bf16>(e);
                }
            l[j] = l[j] * alpha[j] + sum;
        }
        if (!fixed && !__all(alpha[0] == 1.0f && alpha[1] == 1.0f)) {
#pragma unroll
            for (int d = 0; d < DVT; ++d) {
                o[d][0] *= alpha[0];
                o[d][1] *= alpha[1];
            }
        }
#pragma unroll
        for (int k = 0; k < 2; ++k)
#pragma unroll
            for (int d = 0; d < DVT; ++d) {
                const typename M::frag fv = load_columns<BF16Elem>(Vs, LPV, k * 32 + lq * 4, k * 32 + 16 + lq * 4, d * 16, l16);
                o[d][0] = M::mac(fv, fp[k][0], o[d][0]);
                o[d][1] = M::mac(fv, fp[k][1], o[d][1]);
            }
    }
#pragma unroll
    for (int j = 0; j < 2; ++j) {
        l[j] += __shfl_xor(l[j], 16);
        l[j] += __shfl_xor(l[j], 32);
        const float inv = 1.0f / l[j];
        const int t = t0 + wave * kRowsPerWave + j * 16 + l16;
        if (t >= nq) continue;
        uint16_t* out = static_cast<uint16_t*>(p.out) + ((row0 + static_cast<int64_t>(t)) * p.heads + h) * p.vdim;
#pragma unroll
        for (int d = 0; d < DVT; ++d) {
            const int c = d * 16 + lq * 4;
            if (p.vdim % 4 == 0) {
                if (c < p.vdim)
                    *reinterpret_cast<u32x2_t*>(out + c) = u32x2_t{pack_bf16(o[d][j][0] * inv, o[d][j][1] * inv), pack_bf16(o[d][j][2] * inv, o[d][j][3] * inv)};
            } else {
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (c + r < p.vdim) out[c + r] = f32_to_bf16_bits(o[d][j][r] * inv);
            }
        }
    }
}

template <typename Elem, int DKT, int DVT>
int launch_paged(const AttnProblem& p, int n_seqs, int max_q, int splits, float* part_o, float* part_ml, int64_t T, hipStream_t s) {
    const size_t lds = paged_lds<Elem>(DVT);
    int rc = allow_lds(reinterpret_cast<const void*>(attn_paged_kernel<Elem, DKT, DVT>), lds);
    if (rc != 0) return rc;
    const dim3 grid(static_cast<unsigned>(ceil_div(static_cast<int64_t>(max_q) * (p.heads / p.kv_heads), 16)),
                    static_cast<unsigned>(n_seqs * p.kv_heads), static_cast<unsigned>(splits));
    launch((attn_paged_kernel<Elem, DKT, DVT>), grid, dim3(256), lds, s, p, splits, part_o, part_ml);
    rc = launch_status();
    if (rc != 0 || splits == 1) return rc;
    launch((attn_combine_kernel<Elem>), dim3(static_cast<unsigned>(T * p.heads)), dim3(kWave), 0, s, part_o, part_ml, splits, p.vdim,
           static_cast<typename Elem::storage*>(p.out));
    return launch_status();
}

template <typename Elem, int DKT>
int values_paged(const AttnProblem& p, int n_seqs, int max_q, int splits, float* part_o, float* part_ml, int64_t T, hipStream_t s) {
    if (p.vdim <= 64) return launch_paged<Elem, DKT, 4>(p, n_seqs, max_q, splits, part_o, part_ml, T, s);
    if (p.vdim <= 128) return launch_paged<Elem, DKT, 8>(p, n_seqs, max_q, splits, part_o, part_ml, T, s);
    return launch_paged<Elem, DKT, 16>(p, n_seqs, max_q, splits, part_o, part_ml, T, s);
}

template <typename Elem>
int keys_paged(const AttnProblem& p, int n_seqs, int max_q, int splits, float* part_o, float* part_ml, int64_t T, hipStream_t s) {
    if (p.dim <= 64) return values_paged<Elem, 2>(p, n_seqs, max_q, splits, part_o, part_ml, T, s);
    if (p.dim <= 128) return values_paged<Elem, 4>(p, n_seqs, max_q, splits, part_o, part_ml, T, s);
    return values_paged<Elem, 8>(p, n_seqs, max_q, splits, part_o, part_ml, T, s);
}

template <int DKT>
int launch_prompt(const AttnProblem& p, int n_seqs, int max_q, hipStream_t s) {
    const dim3 grid(static_cast<unsigned>(p.heads), static_cast<unsigned>(ceil_div(max_q, kRows)), static_cast<unsigned>(n_seqs));
    if (p.vdim <= 64) launch((attn_prompt_kernel<DKT, 4>), grid, dim3(256), 0, s, p);
    else launch((attn_prompt_kernel<DKT, 8>), grid, dim3(256), 0, s, p);
    return launch_status();
}

}  // namespace

bool attn_supported(int heads, int kv_heads, int dim, int vdim, int rot) {
    return heads > 0 && heads <= 65535 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && dim <= 256 && vdim > 0 && vdim <= 256 &&
           rot >= 0 && rot % 2 == 0 && rot <= dim;
}

int launch_attn_prepare(const AttnProblem& p, int64_t T, hipStream_t s) {
    const dim3 grid(static_cast<unsigned>(T), T <= 256 ? static_cast<unsigned>(ceil_div(p.heads + p.kv_heads, 4)) : 1u);
    const size_t lds = sizeof(float) * (p.rot > 0 ? p.rot : 1);
    const size_t two = 2 * (p.dtype == EM_DTYPE_BF16 ? 2 : 4);
    const bool pair = p.dim % 2 == 0 && p.stride % 2 == 0 && reinterpret_cast<uintptr_t>(p.q) % two == 0 && reinterpret_cast<uintptr_t>(p.k) % two == 0;
    if (p.dtype == EM_DTYPE_BF16) {
        if (pair) launch((attn_prepare_kernel<BF16Elem, true>), grid, dim3(256), lds, s, p);
        else launch((attn_prepare_kernel<BF16Elem, false>), grid, dim3(256), lds, s, p);
    } else {
        if (pair) launch((attn_prepare_kernel<F32Elem, true>), grid, dim3(256), lds, s, p);
        else launch((attn_prepare_kernel<F32Elem, false>), grid, dim3(256), lds, s, p);
    }
    return launch_status();
}

int launch_attn_paged(const AttnProblem& p, int n_seqs, int max_q, int splits, float* part_o, float* part_ml, int64_t T, hipStream_t s) {
    return p.dtype == EM_DTYPE_BF16 ? keys_paged<BF16Elem>(p, n_seqs, max_q, splits, part_o, part_ml, T, s)
                                    : keys_paged<F32Elem>(p, n_seqs, max_q, splits, part_o, part_ml, T, s);
}

// registers bound the size of the values
bool attn_prompt_supported(int dim, int vdim) { return dim > 0 && dim <= 256 && vdim > 0 && vdim <= 128; }

int launch_attn_prompt(const AttnProblem& p, int n_seqs, int max_q, hipStream_t s) {
    if (p.dim <= 64) return launch_prompt<2>(p, n_seqs, max_q, s);
    if (p.dim <= 96) return launch_prompt<3>(p, n_seqs, max_q, s);
    if (p.dim <= 128) return launch_prompt<4>(p, n_seqs, max_q, s);
    return launch_prompt<8>(p, n_seqs, max_q, s);
}

}  // namespace em
