// Latent attention over a paged cache that holds, per token, the normed latent c and one rotated key part shared by
// all heads.
//
// A head's key is W_uk c, its value W_uv c.  Over the cache the up-projections are moved to the other side of the dot
// products: q_lat = W_uk^T q per head, score = (q_lat . c + q_rot . k_rot) * scale, and the head's output is
// W_uv (sum p c): every head reads the same cached row, once.  launch_head_gemm makes both small products.
#include "decoder.h"
#include "mma.h"

namespace em {
namespace {

// ---- norm of the latent, rotation, cache write ----
template <typename Elem>
__global__ __launch_bounds__(256) void latent_prepare_kernel(LatentProblem p) {
    typedef typename Elem::storage S;
    extern __shared__ float cs[];  // [rot / 2] cosines, [rot / 2] sines
    __shared__ float wave_sum[4];
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x, half = p.rot / 2;
    const float pos = static_cast<float>(p.positions[t]);
    for (int i = tid; i < half; i += 256) {
        float sn, c;
        sincosf(pos * p.inv_freq[i], &sn, &c);
        cs[i] = c;
        cs[half + i] = sn;
    }
    const S* d = static_cast<const S*>(p.down) + t * p.down_stride;
    float sum = 0.0f;
    for (int i = tid; i < p.rank; i += 256) {
        const float v = Elem::load(d[i]);
        sum = fmaf(v, v, sum);
    }
#pragma unroll
    for (int off = kWave / 2; off > 0; off >>= 1) sum += __shfl_xor(sum, off);
    if ((tid & 63) == 0) wave_sum[tid >> 6] = sum;
    __syncthreads();
    const float rms = sqrtf((wave_sum[0] + wave_sum[1] + wave_sum[2] + wave_sum[3]) / static_cast<float>(p.rank) + p.eps);
    const int pitch = latent_pitch(p.rank), row = latent_row_elems(p.rank, p.rot);
    S* c = static_cast<S*>(p.cache) + static_cast<int64_t>(p.cache_rows[t]) * row;
    for (int i = tid; i < pitch; i += 256) c[i] = Elem::store(i < p.rank ? Elem::load(d[i]) / rms * p.latent_w[i] : 0.0f);
    for (int i = tid; i < row - pitch; i += 256) {
        float v = 0.0f;
        if (i < p.rot) {
            const int j = i < half ? i : i - half;
            const float a = Elem::load(d[p.rank + j]), b = Elem::load(d[p.rank + half + j]);
            v = i < half ? a * cs[j] - b * cs[half + j] : b * cs[j] + a * cs[half + j];
        }
        c[pitch + i] = Elem::store(v);
    }
    S* q = static_cast<S*>(p.q) + t * p.q_stride;
    for (int i = tid; i < p.heads * half; i += 256) {
        const int h = i / half, j = i - h * half;
        S* qr = q + h * (p.dim + p.rot) + p.dim;
        const float a = Elem::load(qr[j]), b = Elem::load(qr[half + j]);
        qr[j] = Elem::store(a * cs[j] - b * cs[half + j]);
        qr[half + j] = Elem::store(b * cs[j] + a * cs[half + j]);
    }
}

// ---- per-head product  out[t, h, n] = sum_k a[t, h, k] b[h][n][k],  b's rows padded with zeros to 32 elements ----
// A wave makes MT * 16 rows by 64 columns.  KSPLIT: the workgroup's four waves make the same tile, each from a quarter of
// the k steps, and add up in LDS (few tiles of long rows); else they stand side by side along the columns.
template <typename Elem, int MT, bool KSPLIT>
__global__ __launch_bounds__(256) void head_gemm_kernel(const typename Elem::storage* __restrict__ a, int64_t a_row,
                                                        int64_t a_head, const typename Elem::storage* __restrict__ b,
                                                        typename Elem::storage* __restrict__ out, int64_t o_row,
                                                        int64_t o_head, int64_t T, int N, int K, bool vec) {
    typedef Mma<Elem> M;
    constexpr int NT = 4;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, lq = lane >> 4;
    const int h = blockIdx.z;
    const int64_t t0 = static_cast<int64_t>(blockIdx.x) * 16 * MT;
    const int n0 = KSPLIT ? blockIdx.y * 64 : blockIdx.y * (blockDim.x / kWave) * 64 + wave * 64;
    if (!KSPLIT && n0 >= N) return;
    const int KP = (K + 31) / 32 * 32;
    const int k_begin = KSPLIT ? KP / 32 * wave / 4 * 32 : 0, k_end = KSPLIT ? KP / 32 * (wave + 1) / 4 * 32 : KP;
    const typename Elem::storage* bh = b + static_cast<int64_t>(h) * N * KP;
    f32x4_t acc[MT][NT];
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int n = 0; n < NT; ++n) acc[m][n] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
    constexpr int kSteps = MT == 4 ? 2 : 4;  // k steps whose operands are in flight together
    for (int k0 = k_begin; k0 < k_end; k0 += 32 * kSteps) {
        typename M::frag fa[kSteps][MT], fb[kSteps][NT];
#pragma unroll
        for (int u = 0; u < kSteps; ++u) {
            const int k = k0 + u * 32 + lq * 8;
            if (k0 + u * 32 < k_end) {
#pragma unroll
                for (int m = 0; m < MT; ++m) {
                    const int64_t t = t0 + m * 16 + l16;
                    fa[u][m] = t < T ? load_frag<Elem>(a + t * a_row + h * a_head + k, K - k, vec) : M::zero();
                }
#pragma unroll
                for (int n = 0; n < NT; ++n) {
                    const int col = n0 + n * 16 + l16;
                    fb[u][n] = col < N ? M::load(bh + static_cast<int64_t>(col) * KP + k) : M::zero();
                }
            }
        }
#pragma unroll
        for (int u = 0; u < kSteps; ++u)
            if (k0 + u * 32 < k_end) {
#pragma unroll
                for (int m = 0; m < MT; ++m)
#pragma unroll
                    for (int n = 0; n < NT; ++n) acc[m][n] = M::mac(fa[u][m], fb[u][n], acc[m][n]);
            }
    }
    if (KSPLIT) {
        __shared__ float red[4][MT * 16 * 64];
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int n = 0; n < NT; ++n)
#pragma unroll
                for (int r = 0; r < 4; ++r) red[wave][(m * 16 + lq * 4 + r) * 64 + n * 16 + l16] = acc[m][n][r];
        __syncthreads();
        for (int i = threadIdx.x; i < MT * 16 * 64; i += 256) {
            const int64_t t = t0 + i / 64;
            const int col = n0 + i % 64;
            if (t < T && col < N) out[t * o_row + h * o_head + col] = Elem::store(red[0][i] + red[1][i] + red[2][i] + red[3][i]);
        }
        return;
    }
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int n = 0; n < NT; ++n)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int64_t t = t0 + m * 16 + lq * 4 + r;
                const int col = n0 + n * 16 + l16;
                if (t < T && col < N) out[t * o_row + h * o_head + col] = Elem::store(acc[m][n][r]);
            }
}

// Rows row0 .. row0 + 7 of column col0 + l16 of an LDS matrix: the second operand's fragment of a matrix that lies with
// its k dimension across rows.
template <typename Elem>
__device__ __forceinline__ typename Mma<Elem>::frag load_transposed(const typename Elem::storage* m, int pitch, int row0,
                                                                    int col0, int l16);
template <>
__device__ __forceinline__ f32x8_t load_transposed<F32Elem>(const float* m, int pitch, int row0, int col0, int l16) {
    f32x8_t f;
#pragma unroll
    for (int i = 0; i < 8; ++i) f[i] = m[(row0 + i) * pitch + col0 + l16];
    return f;
}
template <>
__device__ __forceinline__ bf16x8_t load_transposed<BF16Elem>(const uint16_t* m, int pitch, int row0, int col0, int l16) {
    // ds_read_b64_tr_b16: the 16 lanes of a group name the four-element pieces of a 4 x 16 block, row by row, and lane i
    // receives column i of it
    typedef short s16x4_t __attribute__((ext_vector_type(4)));
    typedef __attribute__((address_space(3))) s16x4_t* lds_ptr;
    const uint16_t* a = m + (row0 + (l16 >> 2)) * pitch + col0 + (l16 & 3) * 4;
    const s16x4_t lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)(a));
    const s16x4_t hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)(a + 4 * pitch));
    bf16x8_t f;
    __builtin_memcpy(&f, &lo, 8);
    __builtin_memcpy(reinterpret_cast<char*>(&f) + 8, &hi, 8);
    return f;
}

// ---- attention over the pages ----
// A workgroup takes 16 (token, head) rows of one sequence, heads fastest, and one of `splits` ranges of their keys.
// Per tile of 32 keys: the tile goes through registers into LDS (the next one is fetched while this one is used), the
// four waves split the score product over key halves and channel halves, 16 threads per row keep the row's running
// maximum and sum, and for the values (the latents again) each wave owns a quarter of the latent's columns.
constexpr int kKeys = 32;
constexpr int kMaxSplits = kLatentMaxSplits;

template <typename Elem> struct LdsPad { static constexpr int n = 16 / sizeof(typename Elem::storage); };

// NTW: 16-column tiles of the latent per wave (rank <= 64 * NTW)
template <typename Elem, int NTW>
__global__ __launch_bounds__(256) void latent_paged_kernel(LatentProblem p, int splits, float* __restrict__ part_o,
                                                           float* __restrict__ part_ml) {
    typedef typename Elem::storage S;
    typedef Mma<Elem> M;
    constexpr int kFetch = NTW + 2;      // 8-element pieces of a key tile per thread
    const int seq = blockIdx.y, split = blockIdx.z;
    const int q0 = p.q_begin[seq], nq = p.q_begin[seq + 1] - q0;
    const int rows = nq * p.heads, r0 = blockIdx.x * 16;
    if (r0 >= rows) return;
    const int start = p.starts[seq];
    const int last = min(r0 + 15, rows - 1) / p.heads;             // last token of this workgroup's rows
    const int n_keys = start + last + 1;
    const int n_tiles = (n_keys + kKeys - 1) / kKeys;
    const int per_split = (n_tiles + splits - 1) / splits;
    const int tile0 = split * per_split, tile1 = min(tile0 + per_split, n_tiles);

    const int pitch_c = latent_pitch(p.rank), row_elems = latent_row_elems(p.rank, p.rot);
    const int DK = (row_elems + 31) / 32 * 32, LP = DK + LdsPad<Elem>::n;
    extern __shared__ __attribute__((aligned(16))) uint8_t lds_raw[];
    S* Qs = reinterpret_cast<S*>(lds_raw);              // [16][LP]
    S* Ks = Qs + 16 * LP;                               // [32][LP]
    constexpr int PP = kKeys + LdsPad<Elem>::n;
    S* Pm = Ks + kKeys * LP;                            // [16][PP]
    float* Sc = reinterpret_cast<float*>(Pm + 16 * PP); // [2][16][33]
    float* Al = Sc + 2 * 16 * 33;                       // [16]
    int* Kr = reinterpret_cast<int*>(Al + 16);          // [2][32] cache row of every key of a tile, -1: no key

    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lq = lane >> 4;
    const int pieces = row_elems / 8;                   // per key

    // queries: [latent | rotated], zeros behind; the same columns of the key rows
    const bool rot_vec = p.rot % 8 == 0 && p.dim % 8 == 0 && p.q_stride % 8 == 0;
    for (int i = tid; i < 16 * (DK / 8); i += 256) {
        const int r = i / (DK / 8), c = (i - r * (DK / 8)) * 8;
        typename M::frag f = M::zero();
        if (r0 + r < rows) {
            const int t = (r0 + r) / p.heads, h = (r0 + r) - t * p.heads;
            const int64_t row = q0 + t;
            if (c < pitch_c) {
                f = load_frag<Elem>(static_cast<const S*>(p.q_latent) + (row * p.heads + h) * pitch_c + c, p.rank - c, true);
            } else if (c < row_elems) {
                f = load_frag<Elem>(static_cast<const S*>(p.q) + row * p.q_stride + h * (p.dim + p.rot) + p.dim + (c - pitch_c),
                                    p.rot - (c - pitch_c), rot_vec);
            }
        }
        store_frag<Elem>(Qs + r * LP + c, f);
    }
    for (int i = tid; i < kKeys * ((DK - row_elems) / 8); i += 256) {
        const int w = (DK - row_elems) / 8, r = i / w;
        store_frag<Elem>(Ks + r * LP + row_elems + (i - r * w) * 8, M::zero());
    }

    // pieces of a key tile that this thread moves
    int pk[kFetch], pc[kFetch];
#pragma unroll
    for (int i = 0; i < kFetch; ++i) {
        const int e = tid + i * 256;
        pk[i] = e / pieces;
        pc[i] = (e - pk[i] * pieces) * 8;
    }
    const int32_t* table = p.tables + static_cast<int64_t>(seq) * p.table_width;
    const S* cache = static_cast<const S*>(p.cache);
    typename M::frag fetched[kFetch];
    auto find_rows = [&](int tile) {
        if (tid < kKeys && tile < tile1) {
            const int key = tile * kKeys + tid, blk = key / p.block_size;
            Kr[(tile & 1) * kKeys + tid] = key < n_keys ? table[blk] * p.block_size + (key - blk * p.block_size) : -1;
        }
    };
    auto fetch = [&](int tile) {
#pragma unroll
        for (int i = 0; i < kFetch; ++i) {
            fetched[i] = M::zero();
            if (pk[i] < kKeys) {
                const int row = Kr[(tile & 1) * kKeys + pk[i]];
                if (row >= 0) fetched[i] = M::load(cache + static_cast<int64_t>(row) * row_elems + pc[i]);
            }
        }
    };

    f32x4_t o[NTW];
#pragma unroll
    for (int n = 0; n < NTW; ++n) o[n] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
    // softmax state of row tid / 16, the same in its 16 threads
    const int srow = tid >> 4, scol = tid & 15;
    const int spos = start + min(r0 + srow, rows - 1) / p.heads;
    float m = -INFINITY, l = 0.0f;

    find_rows(tile0);
    find_rows(tile0 + 1);
    __syncthreads();
    if (tile0 < tile1) fetch(tile0);
    for (int tile = tile0; tile < tile1; ++tile) {
        __syncthreads();   // the previous tile has been used (and, the first time, Qs is written)
#pragma unroll
        for (int i = 0; i < kFetch; ++i)
            if (pk[i] < kKeys) store_frag<Elem>(Ks + pk[i] * LP + pc[i], fetched[i]);
        if (tile + 1 < tile1) fetch(tile + 1);
        __syncthreads();
        find_rows(tile + 2);     // into the half that this tile's rows leave; read behind the next barriers
        {
            f32x4_t s = {0.0f, 0.0f, 0.0f, 0.0f};
            const S* qp = Qs + l16 * LP + lq * 8;
            const S* kp = Ks + ((wave & 1) * 16 + l16) * LP + lq * 8;
            for (int k = (wave >> 1) * 32; k < DK; k += 64) s = M::mac(M::load(qp + k), M::load(kp + k), s);
#pragma unroll
            for (int r = 0; r < 4; ++r) Sc[((wave >> 1) * 16 + lq * 4 + r) * 33 + (wave & 1) * 16 + l16] = s[r];
        }
        __syncthreads();
        {
            const float* s0 = Sc + srow * 33;
            const float* s1 = s0 + 16 * 33;
            float sv[2], mx = -INFINITY;
#pragma unroll
            for (int j = 0; j < 2; ++j) {
                const int c = scol + j * 16;
                sv[j] = tile * kKeys + c <= spos ? (s0[c] + s1[c]) * p.scale : -INFINITY;
                mx = fmaxf(mx, sv[j]);
            }
#pragma unroll
            for (int off = 8; off > 0; off >>= 1) mx = fmaxf(mx, __shfl_xor(mx, off));
            const float mn = fmaxf(m, mx);
            const float alpha = mn == -INFINITY ? 1.0f : expf(m - mn);
            float sum = 0.0f;
#pragma unroll
            for (int j = 0; j < 2; ++j) {
                const float e = sv[j] == -INFINITY ? 0.0f : expf(sv[j] - mn);
                sum += e;
                Pm[srow * PP + scol + j * 16] = Elem::store(e);
            }
#pragma unroll
            for (int off = 8; off > 0; off >>= 1) sum += __shfl_xor(sum, off);
            l = l * alpha + sum;
            m = mn;
            if (scol == 0) Al[srow] = alpha;
        }
        __syncthreads();
        {
            const typename M::frag fp = M::load(Pm + l16 * PP + lq * 8);
            const f32x4_t a4 = *reinterpret_cast<const f32x4_t*>(Al + lq * 4);
#pragma unroll
            for (int n = 0; n < NTW; ++n) {
                const int c = (wave * NTW + n) * 16;
                if (c < pitch_c) {
                    o[n] *= a4;
                    o[n] = M::mac(fp, load_transposed<Elem>(Ks, LP, lq * 8, c, l16), o[n]);
                }
            }
        }
    }
    // per-row sum and maximum to the layout of the accumulators
    __syncthreads();
    float* Lm = Sc;
    if (scol == 0) {
        Lm[srow] = m;
        Lm[16 + srow] = l;
    }
    __syncthreads();
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int rr = lq * 4 + r;
        if (r0 + rr >= rows) continue;
        const int64_t row = static_cast<int64_t>(q0) * p.heads + r0 + rr;
        if (splits == 1) {
            const float mr = Lm[rr], sk = p.sink[(r0 + rr) % p.heads];
            const float top = fmaxf(mr, sk), w = expf(mr - top);
            const float inv = w / (Lm[16 + rr] * w + expf(sk - top));
#pragma unroll
            for (int n = 0; n < NTW; ++n) {
                const int c = (wave * NTW + n) * 16 + l16;
                if (c < pitch_c) static_cast<S*>(p.out)[row * pitch_c + c] = Elem::store(c < p.rank ? o[n][r] * inv : 0.0f);
            }
        } else {
#pragma unroll
            for (int n = 0; n < NTW; ++n) {
                const int c = (wave * NTW + n) * 16 + l16;
                if (c < pitch_c) part_o[(row * splits + split) * pitch_c + c] = o[n][r];
            }
            if (wave == 0 && l16 == 0) {
                part_ml[(row * splits + split) * 2] = Lm[rr];
                part_ml[(row * splits + split) * 2 + 1] = Lm[16 + rr];
            }
        }
    }
}

template <typename Elem>
__global__ __launch_bounds__(128) void latent_combine_kernel(const float* __restrict__ part_o,
                                                             const float* __restrict__ part_ml,
                                                             const float* __restrict__ sink, int heads, int splits,
                                                             int pitch, int rank, typename Elem::storage* __restrict__ out) {
    constexpr int kAhead = 8;
    __shared__ float weight[kMaxSplits];
    const int64_t row = blockIdx.x;
    const float* ml = part_ml + row * splits * 2;
    const float sk = sink[row % heads];
    float top = sk;
    for (int s = 0; s < splits; ++s) top = fmaxf(top, ml[2 * s]);
    float den = expf(sk - top);
    for (int s = 0; s < splits; ++s) den += ml[2 * s + 1] * expf(ml[2 * s] - top);
    for (int s = threadIdx.x; s < splits; s += 128) weight[s] = expf(ml[2 * s] - top) / den;
    __syncthreads();
    for (int c = threadIdx.x * 4; c < pitch; c += 512) {   // pitch is a multiple of eight
        const f32x4_t* src = reinterpret_cast<const f32x4_t*>(part_o + row * splits * pitch + c);
        f32x4_t v = {0.0f, 0.0f, 0.0f, 0.0f};
        for (int s0 = 0; s0 < splits; s0 += kAhead) {
            f32x4_t x[kAhead];
#pragma unroll
            for (int j = 0; j < kAhead; ++j)
                x[j] = s0 + j < splits ? src[static_cast<int64_t>(s0 + j) * pitch / 4] : f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int j = 0; j < kAhead; ++j)
                if (s0 + j < splits) v += x[j] * weight[s0 + j];
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) out[row * pitch + c + j] = Elem::store(c + j < rank ? v[j] : 0.0f);
    }
}

// cached rows of every sequence, copied behind each other (sequence s at row k_begin[s]; rows up to k_begin[s + 1] that
// hold no key are zero)
template <typename Elem>
__global__ __launch_bounds__(256) void latent_gather_kernel(const typename Elem::storage* __restrict__ cache,
                                                            const int32_t* __restrict__ tables, int table_width,
                                                            int block_size, const int32_t* __restrict__ k_begin,
                                                            const int32_t* __restrict__ k_lens, int row_elems,
                                                            typename Elem::storage* __restrict__ out) {
    const int seq = blockIdx.y, pieces = row_elems / 8;
    const int64_t e = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
    const int key = static_cast<int>(e / pieces), c = static_cast<int>(e - static_cast<int64_t>(key) * pieces) * 8;
    if (key >= k_begin[seq + 1] - k_begin[seq]) return;
    typename Mma<Elem>::frag f = Mma<Elem>::zero();
    if (key < k_lens[seq]) {
        const int blk = key / block_size;
        const int64_t row = static_cast<int64_t>(tables[static_cast<int64_t>(seq) * table_width + blk]) * block_size + key % block_size;
        f = Mma<Elem>::load(cache + row * row_elems + c);
    }
    store_frag<Elem>(out + static_cast<int64_t>(k_begin[seq] + key) * row_elems + c, f);
}

template <typename Elem, int NTW>
int launch_paged(const LatentProblem& p, int n_seqs, int max_q, int splits, float* part_o, float* part_ml, hipStream_t s) {
    typedef typename Elem::storage S;
    const int DK = static_cast<int>(round_up(latent_row_elems(p.rank, p.rot), 32)), LP = DK + LdsPad<Elem>::n;
    const size_t lds = sizeof(S) * (48 * LP + 16 * (kKeys + LdsPad<Elem>::n)) + sizeof(float) * (2 * 16 * 33 + 16 + 2 * kKeys);
    const int rc = allow_lds(reinterpret_cast<const void*>(latent_paged_kernel<Elem, NTW>), lds);
    if (rc != 0) return rc;
    const dim3 grid(static_cast<unsigned>(ceil_div(static_cast<int64_t>(max_q) * p.heads, 16)), static_cast<unsigned>(n_seqs),
                    static_cast<unsigned>(splits));
    launch((latent_paged_kernel<Elem, NTW>), grid, dim3(256), lds, s, p, splits, part_o, part_ml);
    return launch_status();
}

template <typename Elem>
int dispatch_paged(const LatentProblem& p, int n_seqs, int max_q, int splits, float* part_o, float* part_ml, int64_t T,
                   hipStream_t s) {
    int rc;
    if (p.rank <= 128) rc = launch_paged<Elem, 2>(p, n_seqs, max_q, splits, part_o, part_ml, s);
    else if (p.rank <= 256) rc = launch_paged<Elem, 4>(p, n_seqs, max_q, splits, part_o, part_ml, s);
    else rc = launch_paged<Elem, 8>(p, n_seqs, max_q, splits, part_o, part_ml, s);
    if (rc != 0 || splits == 1) return rc;
    launch((latent_combine_kernel<Elem>), dim3(static_cast<unsigned>(T * p.heads)), dim3(128), 0, s, part_o, part_ml, p.sink,
           p.heads, splits, latent_pitch(p.rank), p.rank, static_cast<typename Elem::storage*>(p.out));
    return launch_status();
}

template <typename Elem>
int head_gemm(const void* a, int64_t a_row, int64_t a_head, const void* b, void* out, int64_t o_row, int64_t o_head,
              int64_t T, int heads, int N, int K, hipStream_t s) {
    typedef typename Elem::storage S;
    const bool vec = a_row % 8 == 0 && a_head % 8 == 0 && reinterpret_cast<uintptr_t>(a) % (8 * sizeof(S)) == 0;
    // as many rows per workgroup as leave the chip filled
    const int64_t cols = ceil_div(N, 64);
    const int mt = ceil_div(T, 64) * cols * heads >= 512 ? 4 : T > 16 && ceil_div(T, 32) * cols * heads >= 256 ? 2 : 1;
    const int64_t wave_tiles = ceil_div(T, 16 * mt) * cols * heads;
    const int waves = static_cast<int>(wave_tiles >= 1024 ? (cols < 4 ? cols : 4) : 1);
    const bool ksplit = waves == 1 && mt == 1 && K >= 256;
    const dim3 grid(static_cast<unsigned>(ceil_div(T, 16 * mt)), static_cast<unsigned>(ceil_div(N, waves * 64)),
                    static_cast<unsigned>(heads)), block(static_cast<unsigned>(ksplit ? 256 : waves * kWave));
#define EM_HEAD_GEMM(MT, KS)                                                                                              \
    launch((head_gemm_kernel<Elem, MT, KS>), grid, block, 0, s, static_cast<const S*>(a), a_row, a_head,                  \
           static_cast<const S*>(b), static_cast<S*>(out), o_row, o_head, T, N, K, vec)
    if (ksplit) EM_HEAD_GEMM(1, true);
    else if (mt == 4) EM_HEAD_GEMM(4, false);
    else if (mt == 2) EM_HEAD_GEMM(2, false);
    else EM_HEAD_GEMM(1, false);
#undef EM_HEAD_GEMM
    return launch_status();
}

}  // namespace

bool latent_supported(int heads, int dim, int rot, int rank) {
    // key rows of one tile per thread: 8-element pieces, at most NTW + 2 of them (see latent_paged_kernel)
    return heads > 0 && heads <= 1024 && dim > 0 && rot >= 0 && rot % 2 == 0 && rot <= 128 && rank > 0 && rank <= 512;
}

int launch_latent_prepare(const LatentProblem& p, int64_t T, hipStream_t s) {
    const dim3 grid(static_cast<unsigned>(T));
    const size_t lds = sizeof(float) * (p.rot > 0 ? p.rot : 1);
    if (p.dtype == EM_DTYPE_BF16) launch((latent_prepare_kernel<BF16Elem>), grid, dim3(256), lds, s, p);
    else launch((latent_prepare_kernel<F32Elem>), grid, dim3(256), lds, s, p);
    return launch_status();
}

int launch_latent_paged(const LatentProblem& p, int n_seqs, int max_q, int splits, float* part_o, float* part_ml,
                        int64_t T, hipStream_t s) {
    return p.dtype == EM_DTYPE_BF16 ? dispatch_paged<BF16Elem>(p, n_seqs, max_q, splits, part_o, part_ml, T, s)
                                    : dispatch_paged<F32Elem>(p, n_seqs, max_q, splits, part_o, part_ml, T, s);
}

int launch_head_gemm(const void* a, int64_t a_row, int64_t a_head, const void* b, void* out, int64_t o_row,
                     int64_t o_head, int64_t T, int heads, int N, int K, int dtype, hipStream_t s) {
    return dtype == EM_DTYPE_BF16 ? head_gemm<BF16Elem>(a, a_row, a_head, b, out, o_row, o_head, T, heads, N, K, s)
                                  : head_gemm<F32Elem>(a, a_row, a_head, b, out, o_row, o_head, T, heads, N, K, s);
}

int launch_latent_gather(const void* cache, const int32_t* tables, int table_width, int block_size, const int32_t* k_begin,
                         const int32_t* k_lens, int n_seqs, int max_k, int row_elems, void* out, int dtype, hipStream_t s) {
    const dim3 grid(static_cast<unsigned>(ceil_div(static_cast<int64_t>(max_k) * (row_elems / 8), 256)), static_cast<unsigned>(n_seqs));
    if (dtype == EM_DTYPE_BF16)
        launch((latent_gather_kernel<BF16Elem>), grid, dim3(256), 0, s, static_cast<const uint16_t*>(cache), tables,
               table_width, block_size, k_begin, k_lens, row_elems, static_cast<uint16_t*>(out));
    else
        launch((latent_gather_kernel<F32Elem>), grid, dim3(256), 0, s, static_cast<const float*>(cache), tables,
               table_width, block_size, k_begin, k_lens, row_elems, static_cast<float*>(out));
    return launch_status();
}

}  // namespace em
