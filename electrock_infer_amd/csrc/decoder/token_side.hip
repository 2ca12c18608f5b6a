// A per-layer token input.  token_gate_kernel is the gate product with its epilogue,
//     g[t] = gelu_tanh(gate x_t) * side[token_t],
// spread over as many workgroups as there are 16 x 16 tiles of g: what decoding needs.  token_side_kernel is the end of a
// layer in one launch (bf16), for prompts, where there are rows enough to fill the chip with 16 each:
//     x <- x + y / rms(y) * post_w                       (the feed-forward's result)
//     g  = gelu_tanh(gate x) * side[token]
//     x <- x + p / rms(p) * side_norm,  p = proj g
//     out = x / rms(x) * next_w, or x                    (what the next layer reads)
// A workgroup takes up to 16 rows of the float32 stream.  A row belongs to one wave in the element-wise phases (its sums
// are wave reductions, no barriers); in between, the rows' bf16 copy in LDS is the first operand of the gate product,
// whose k range the eight waves share out, and p, rounded to bf16, takes that copy's place for the last phase.
#include "decoder.h"
#include "mma.h"

namespace em {
namespace {

constexpr int kThreads = 512;
constexpr int kWaves = kThreads / kWave;
constexpr int kTileRows = 16;
constexpr int kGateTiles = 4;  // 16-column tiles of the gate product that a wave accumulates at a time

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int off = kWave / 2; off > 0; off >>= 1) v += __shfl_xor(v, off);
    return v;
}

__device__ __forceinline__ void load4(const uint16_t* p, float (&v)[4]) {
    const u32x2_t w = *reinterpret_cast<const u32x2_t*>(p);
    v[0] = bf16_lo(w[0]);
    v[1] = bf16_hi(w[0]);
    v[2] = bf16_lo(w[1]);
    v[3] = bf16_hi(w[1]);
}
__device__ __forceinline__ void store4(uint16_t* p, const float (&v)[4]) {
    *reinterpret_cast<u32x2_t*>(p) = u32x2_t{pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3])};
}

// One workgroup per 16 x 16 tile of g; its waves share out the k range.
template <typename Elem>
__global__ __launch_bounds__(kThreads) void token_gate_kernel(const typename Elem::storage* __restrict__ x,
                                                              const typename Elem::storage* __restrict__ gate,
                                                              const int32_t* __restrict__ tokens,
                                                              const typename Elem::storage* __restrict__ table,
                                                              int64_t table_stride, int column0,
                                                              typename Elem::storage* __restrict__ g, int64_t T, int W, int dim) {
    typedef Mma<Elem> M;
    constexpr int kAhead = 4;
    __shared__ float part[kWaves][256];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lq = lane >> 4;
    const int64_t t0 = static_cast<int64_t>(blockIdx.x) * 16;
    const int d0 = blockIdx.y * 16;
    const int steps = (W + 31) / 32;
    const bool vec = W % 8 == 0, row_ok = t0 + l16 < T, col_ok = d0 + l16 < dim;
    const typename Elem::storage* xr = x + (row_ok ? t0 + l16 : t0) * W;
    const typename Elem::storage* wr = gate + static_cast<int64_t>(col_ok ? d0 + l16 : d0) * W;  // (extra columns are not stored)
    f32x4_t acc = {0.0f, 0.0f, 0.0f, 0.0f};
    for (int s = wave; s < steps; s += kWaves * kAhead) {
        typename M::frag fx[kAhead], fw[kAhead];
#pragma unroll
        for (int u = 0; u < kAhead; ++u)
            if (s + u * kWaves < steps) {
                const int k = (s + u * kWaves) * 32 + lq * 8;
                fx[u] = load_frag<Elem>(xr + k, W - k, vec);
                fw[u] = load_frag<Elem>(wr + k, W - k, vec);
            }
#pragma unroll
        for (int u = 0; u < kAhead; ++u)
            if (s + u * kWaves < steps) acc = M::mac(fx[u], fw[u], acc);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) part[wave][(lq * 4 + r) * 16 + l16] = acc[r];
    __syncthreads();
    if (tid < 256) {
        const int r = tid >> 4, d = d0 + (tid & 15);
        if (t0 + r < T && d < dim) {
            float z = 0.0f;
#pragma unroll
            for (int w = 0; w < kWaves; ++w) z += part[w][tid];
            const float e = Elem::load(table[static_cast<int64_t>(tokens[t0 + r]) * table_stride + column0 + d]);
            g[(t0 + r) * dim + d] = Elem::store(gelu_tanh(z) * e);
        }
    }
}

// NV: four-element pieces of a row per lane (W <= 256 * NV).  FULL: W % 128 == 0 and dim % 32 == 0, no operand piece is
// ragged and several weight fragments are fetched together.
template <int NV, bool FULL>
__global__ __launch_bounds__(kThreads, NV <= 8 ? 4 : 2) void token_side_kernel(TokenSideProblem p) {
    typedef Mma<BF16Elem> M;
    extern __shared__ __attribute__((aligned(16))) uint8_t lds_raw[];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lq = lane >> 4;
    const int W = p.W, LPX = (W + 31) / 32 * 32 + 8, dim = p.dim, DP = (dim + 31) / 32 * 32, LPG = DP + 8;
    uint16_t* Xs = reinterpret_cast<uint16_t*>(lds_raw);          // [16][LPX] rows in bf16; later p
    float* Part = reinterpret_cast<float*>(lds_raw);              // [8][16][64] partial gate products, in the same place
    uint16_t* Gs = reinterpret_cast<uint16_t*>(lds_raw + p.g_offset);  // [16][LPG]
    const int64_t row0 = static_cast<int64_t>(blockIdx.x) * p.rows_per_group;
    const int n = static_cast<int>(min(static_cast<int64_t>(p.rows_per_group), p.T - row0));
    const float inv_w = 1.0f / static_cast<float>(W);

    // ---- x + normed y, as bf16, into LDS ----
    float y_rstd[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int r = wave + i * kWaves;
        y_rstd[i] = 0.0f;
        if (r < n) {
            const uint16_t* yr = p.y + (row0 + r) * W;
            float y[NV][4], sum = 0.0f;
            f32x4_t x[NV];
#pragma unroll
            for (int j = 0; j < NV; ++j) {
                const int c = (lane + j * 64) * 4;
                if (c < W) {
                    load4(yr + c, y[j]);
                    x[j] = *reinterpret_cast<const f32x4_t*>(p.x + (row0 + r) * W + c);
                }
            }
#pragma unroll
            for (int j = 0; j < NV; ++j)
                if ((lane + j * 64) * 4 < W) {
#pragma unroll
                    for (int e = 0; e < 4; ++e) sum = fmaf(y[j][e], y[j][e], sum);
                }
            y_rstd[i] = 1.0f / sqrtf(wave_sum(sum) * inv_w + p.eps);
#pragma unroll
            for (int j = 0; j < NV; ++j) {
                const int c = (lane + j * 64) * 4;
                if (c < W) {
                    const f32x4_t w4 = *reinterpret_cast<const f32x4_t*>(p.post_w + c);
                    float v[4];
#pragma unroll
                    for (int e = 0; e < 4; ++e) v[e] = x[j][e] + y[j][e] * y_rstd[i] * w4[e];
                    store4(Xs + r * LPX + c, v);
                }
            }
        } else if (r < kTileRows) {
            const float z[4] = {0.0f, 0.0f, 0.0f, 0.0f};
            for (int c = lane * 4; c < W; c += 256) store4(Xs + r * LPX + c, z);
        }
    }
    for (int i = tid; i < kTileRows * (LPX - W); i += kThreads) {   // the columns up to a multiple of 32
        const int w = LPX - W, r = i / w;
        Xs[r * LPX + W + (i - r * w)] = 0;
    }
    for (int i = tid; i < kTileRows * (DP - dim); i += kThreads) {
        const int w = DP - dim, r = i / w;
        Gs[r * LPG + dim + (i - r * w)] = 0;
    }
    // ---- gate product, 64 columns at a time ----
    const int steps = (W + 31) / 32;
    for (int d0 = 0; d0 < dim; d0 += kGateTiles * 16) {
        __syncthreads();
        f32x4_t acc[kGateTiles];
#pragma unroll
        for (int t = 0; t < kGateTiles; ++t) acc[t] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
        if (FULL) {
            constexpr int kAhead = 4;
            for (int s = wave; s < steps; s += kWaves * kAhead) {
                typename M::frag fw[kAhead][kGateTiles];
#pragma unroll
                for (int u = 0; u < kAhead; ++u)
                    if (s + u * kWaves < steps) {
#pragma unroll
                        for (int t = 0; t < kGateTiles; ++t)
                            if (d0 + t * 16 < dim)
                                fw[u][t] = M::load(p.gate + static_cast<int64_t>(d0 + t * 16 + l16) * W + (s + u * kWaves) * 32 + lq * 8);
                    }
#pragma unroll
                for (int u = 0; u < kAhead; ++u)
                    if (s + u * kWaves < steps) {
                        const typename M::frag fx = M::load(Xs + l16 * LPX + (s + u * kWaves) * 32 + lq * 8);
#pragma unroll
                        for (int t = 0; t < kGateTiles; ++t)
                            if (d0 + t * 16 < dim) acc[t] = M::mac(fx, fw[u][t], acc[t]);
                    }
            }
        } else for (int s = wave; s < steps; s += kWaves) {
            const int k = s * 32 + lq * 8;
            const typename M::frag fx = M::load(Xs + l16 * LPX + k);
#pragma unroll
            for (int t = 0; t < kGateTiles; ++t) {
                const int d = d0 + t * 16 + l16;
                // (W is a multiple of four: the last piece of a row may be half)
                if (d0 + t * 16 < dim)
                    acc[t] = M::mac(fx, d < dim ? load_frag<BF16Elem>(p.gate + static_cast<int64_t>(d) * W + k, W - k, W % 8 == 0) : M::zero(), acc[t]);
            }
        }
        // the partial products lie where the rows did: for more columns than one turn takes they lie behind everything
        float* part = p.part_offset == 0 ? Part : reinterpret_cast<float*>(lds_raw + p.part_offset);
        __syncthreads();
#pragma unroll
        for (int t = 0; t < kGateTiles; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) part[(wave * kTileRows + lq * 4 + r) * 64 + t * 16 + l16] = acc[t][r];
        __syncthreads();
        for (int i = tid; i < kTileRows * 64; i += kThreads) {
            const int r = i / 64, d = d0 + i % 64;
            if (d < dim) {
                float z = 0.0f;
#pragma unroll
                for (int w = 0; w < kWaves; ++w) z += part[w * kTileRows * 64 + i];
                float e = 0.0f;
                if (r < n) e = bf16_bits_to_f32(p.table[static_cast<int64_t>(p.tokens[row0 + r]) * p.table_stride + p.column0 + d]);
                Gs[r * LPG + d] = f32_to_bf16_bits(gelu_tanh(z) * e);
            }
        }
    }
    __syncthreads();
    // ---- p = proj g: every wave a share of the columns ----
    const int col_tiles = (W + 15) / 16;
    if (FULL) {
        constexpr int kAhead = 8;  // column tiles whose weights are fetched together
        for (int t = wave; t < col_tiles; t += kWaves * kAhead) {
            f32x4_t acc[kAhead];
#pragma unroll
            for (int u = 0; u < kAhead; ++u) acc[u] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
            for (int k = lq * 8; k < DP; k += 32) {
                typename M::frag fw[kAhead];
#pragma unroll
                for (int u = 0; u < kAhead; ++u)
                    if (t + u * kWaves < col_tiles)
                        fw[u] = M::load(p.proj + static_cast<int64_t>((t + u * kWaves) * 16 + l16) * dim + k);
                const typename M::frag fg = M::load(Gs + l16 * LPG + k);
#pragma unroll
                for (int u = 0; u < kAhead; ++u)
                    if (t + u * kWaves < col_tiles) acc[u] = M::mac(fg, fw[u], acc[u]);
            }
#pragma unroll
            for (int u = 0; u < kAhead; ++u)
                if (t + u * kWaves < col_tiles) {
#pragma unroll
                    for (int r = 0; r < 4; ++r) Xs[(lq * 4 + r) * LPX + (t + u * kWaves) * 16 + l16] = f32_to_bf16_bits(acc[u][r]);
                }
        }
    } else for (int t = wave; t < col_tiles; t += kWaves) {
        const int c = t * 16 + l16;
        f32x4_t acc = {0.0f, 0.0f, 0.0f, 0.0f};
        for (int k = lq * 8; k < DP; k += 32) {
            const typename M::frag fg = M::load(Gs + l16 * LPG + k);
            acc = M::mac(fg, c < W ? load_frag<BF16Elem>(p.proj + static_cast<int64_t>(c) * dim + k, dim - k, dim % 8 == 0) : M::zero(), acc);
        }
        if (c < W) {
#pragma unroll
            for (int r = 0; r < 4; ++r) Xs[(lq * 4 + r) * LPX + c] = f32_to_bf16_bits(acc[r]);
        }
    }
    __syncthreads();
    // ---- the stream and the next layer's input ----
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int r = wave + i * kWaves;
        if (r >= n) continue;
        const int64_t row = row0 + r;
        float sum = 0.0f, x[NV][4], y[NV][4];
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            const int c = (lane + j * 64) * 4;
            if (c < W) {
                load4(p.y + row * W + c, y[j]);
                const f32x4_t x4 = *reinterpret_cast<const f32x4_t*>(p.x + row * W + c);
#pragma unroll
                for (int e = 0; e < 4; ++e) x[j][e] = x4[e];
            }
        }
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            const int c = (lane + j * 64) * 4;
            if (c < W) {
                float v[4];
                load4(Xs + r * LPX + c, v);
#pragma unroll
                for (int e = 0; e < 4; ++e) sum = fmaf(v[e], v[e], sum);
            }
        }
        const float rstd = 1.0f / sqrtf(wave_sum(sum) * inv_w + p.eps);
        sum = 0.0f;
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            const int c = (lane + j * 64) * 4;
            if (c < W) {
                float v[4];
                load4(Xs + r * LPX + c, v);
                const f32x4_t w4 = *reinterpret_cast<const f32x4_t*>(p.post_w + c);
                const f32x4_t s4 = *reinterpret_cast<const f32x4_t*>(p.side_norm + c);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    x[j][e] += y[j][e] * y_rstd[i] * w4[e] + v[e] * rstd * s4[e];
                    sum = fmaf(x[j][e], x[j][e], sum);
                }
            }
        }
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            const int c = (lane + j * 64) * 4;
            if (c < W) *reinterpret_cast<f32x4_t*>(p.x + row * W + c) = f32x4_t{x[j][0], x[j][1], x[j][2], x[j][3]};
        }
        const float x_rstd = p.next_w != nullptr ? 1.0f / sqrtf(wave_sum(sum) * inv_w + p.eps) : 1.0f;
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            const int c = (lane + j * 64) * 4;
            if (c < W) {
                float v[4];
                if (p.next_w != nullptr) {
                    const f32x4_t w4 = *reinterpret_cast<const f32x4_t*>(p.next_w + c);
#pragma unroll
                    for (int e = 0; e < 4; ++e) v[e] = x[j][e] * x_rstd * w4[e];
                } else {
#pragma unroll
                    for (int e = 0; e < 4; ++e) v[e] = x[j][e];
                }
                store4(p.out + row * p.out_stride + c, v);
            }
        }
    }
}

constexpr int kPartBytes = kWaves * kTileRows * 64 * 4;

// LDS: the rows (or, when one turn takes all gate columns, the partial products in their place), the gate's result, and
// the partial products if they need room of their own.
size_t lds_bytes(int W, int dim, int* g_offset, int* part_offset) {
    const int rows = static_cast<int>(round_up(W, 32) + 8) * kTileRows * 2;
    const bool one_turn = dim <= kGateTiles * 16;
    const int first = one_turn && rows < kPartBytes ? kPartBytes : rows;
    *g_offset = first;
    const int g = static_cast<int>(round_up(dim, 32) + 8) * kTileRows * 2;
    *part_offset = one_turn ? 0 : first + g;
    return static_cast<size_t>(first) + g + (one_turn ? 0 : kPartBytes);
}

template <int NV, bool FULL>
int launch_side(const TokenSideProblem& p, size_t lds, hipStream_t s) {
    const int rc = allow_lds(reinterpret_cast<const void*>(token_side_kernel<NV, FULL>), lds);
    if (rc != 0) return rc;
    launch((token_side_kernel<NV, FULL>), dim3(static_cast<unsigned>(ceil_div(p.T, p.rows_per_group))), dim3(kThreads), lds, s, p);
    return launch_status();
}

}  // namespace

int launch_token_gate(const void* x, const void* gate, const int32_t* tokens, const void* table, int64_t table_stride,
                      int column0, void* g, int64_t T, int W, int dim, int dtype, hipStream_t s) {
    const dim3 grid(static_cast<unsigned>(ceil_div(T, 16)), static_cast<unsigned>(ceil_div(dim, 16)));
    if (dtype == EM_DTYPE_BF16)
        launch((token_gate_kernel<BF16Elem>), grid, dim3(kThreads), 0, s, static_cast<const uint16_t*>(x),
               static_cast<const uint16_t*>(gate), tokens, static_cast<const uint16_t*>(table), table_stride, column0,
               static_cast<uint16_t*>(g), T, W, dim);
    else
        launch((token_gate_kernel<F32Elem>), grid, dim3(kThreads), 0, s, static_cast<const float*>(x),
               static_cast<const float*>(gate), tokens, static_cast<const float*>(table), table_stride, column0,
               static_cast<float*>(g), T, W, dim);
    return launch_status();
}

bool token_side_supported(int W, int dim) {
    int a, b;
    return W > 0 && W % 4 == 0 && W <= 4096 && dim > 0 && dim <= 1024 && lds_bytes(W, dim, &a, &b) <= kLdsPerCu;
}

int launch_token_side(TokenSideProblem p, hipStream_t s) {
    const size_t lds = lds_bytes(p.W, p.dim, &p.g_offset, &p.part_offset);
    p.rows_per_group = p.T <= 512 ? 8 : 16;  // one row per wave while the chip is not full
    if (p.W % 128 == 0 && p.dim % 32 == 0) {
        if (p.W <= 1024) return launch_side<4, true>(p, lds, s);
        if (p.W <= 2048) return launch_side<8, true>(p, lds, s);
        return launch_side<16, true>(p, lds, s);
    }
    if (p.W <= 1024) return launch_side<4, false>(p, lds, s);
    if (p.W <= 2048) return launch_side<8, false>(p, lds, s);
    return launch_side<16, false>(p, lds, s);
}

}  // namespace em
