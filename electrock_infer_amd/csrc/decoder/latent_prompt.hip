// Latent attention for long portions of a prompt, bf16: keys and values of every head are written out once by two
// matrix products over the latents of the context (keys [K, heads * dim], values transposed [heads * vdim, K]) and a
// tiled softmax attention runs on them.
//
// A workgroup takes 128 queries of one head, 32 per wave.  Per tile of 64 keys a wave computes S^T = K Q^T: a lane then
// holds, for one query, keys (lane / 16) * 4 + 0..3 of every 16.  Since a sum over keys may run in any order as long as
// both operands agree, these registers, rounded to bf16, are the second operand of O^T = V^T P^T as they are: the values
// only have to lie in LDS in the matching key order.  Nothing of the probabilities goes through LDS, the running maximum
// and sum of a query live in one register of its four lanes, and a lane's results are four neighbouring outputs.
#include "decoder.h"
#include "mma.h"

namespace em {
namespace {

constexpr int kTileKeys = 64;
constexpr int kRowsPerWave = 32;
constexpr int kRows = 4 * kRowsPerWave;
constexpr float kLog2e = 1.4426950408889634f;

// DKT: 32-element steps of dim + rot; DVT: 16-element tiles of vdim
template <int DKT, int DVT>
__global__ __launch_bounds__(256, 2) void latent_prompt_kernel(LatentPromptProblem p) {
    typedef Mma<BF16Elem> M;
    constexpr int LPK = DKT * 32 + 8, LPV = kTileKeys + 8;
    constexpr int kFetchK = kTileKeys * DKT * 4 / 256, kFetchV = DVT * 16 * (kTileKeys / 8) / 256;
    __shared__ __attribute__((aligned(16))) uint16_t Ks[kTileKeys * LPK];
    __shared__ __attribute__((aligned(16))) uint16_t Vs[DVT * 16 * LPV];
    const int h = blockIdx.x, seq = blockIdx.z;
    const int row0 = p.q_begin[seq], nq = p.q_begin[seq + 1] - row0;
    const int t0 = (static_cast<int>(gridDim.y) - 1 - static_cast<int>(blockIdx.y)) * kRows;  // long rows start first
    if (t0 >= nq) return;
    const int start = p.starts[seq];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lq = lane >> 4;
    const int D = p.dim + p.rot;
    const int64_t k0 = p.k_begin[seq];
    const int n_tiles = (start + min(t0 + kRows, nq) + kTileKeys - 1) / kTileKeys;
    const int first_pos = start + t0 + wave * kRowsPerWave;      // of this wave's first query

    typename M::frag fq[2][DKT];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
        const int t = t0 + wave * kRowsPerWave + j * 16 + l16;
        const uint16_t* q = p.q + (row0 + static_cast<int64_t>(min(t, nq - 1))) * p.q_stride + h * D;
#pragma unroll
        for (int k = 0; k < DKT; ++k) {
            const int c = k * 32 + lq * 8;
            fq[j][k] = c < D ? M::load(q + c) : M::zero();
        }
    }

    typename M::frag rk[kFetchK], rv[kFetchV];
    auto fetch = [&](int tile) {
        const int64_t key0 = k0 + static_cast<int64_t>(tile) * kTileKeys;
#pragma unroll
        for (int i = 0; i < kFetchK; ++i) {
            const int e = tid + i * 256, key = e / (DKT * 4), c = (e % (DKT * 4)) * 8;
            rk[i] = M::zero();
            if (c < p.dim) rk[i] = M::load(p.k + (key0 + key) * p.k_stride + h * p.dim + c);
            else if (c < D) rk[i] = M::load(p.k_rot + (key0 + key) * p.k_rot_stride + (c - p.dim));
        }
#pragma unroll
        for (int i = 0; i < kFetchV; ++i) {
            const int e = tid + i * 256, d = e / (kTileKeys / 8), c = (e % (kTileKeys / 8)) * 8;
            rv[i] = d < p.vdim ? M::load(p.vt + (static_cast<int64_t>(h) * p.vdim + d) * p.v_stride + key0 + c) : M::zero();
        }
    };

    f32x4_t o[DVT][2];
#pragma unroll
    for (int d = 0; d < DVT; ++d) o[d][0] = o[d][1] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
    float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.0f, 0.0f};   // m in units of log2; l: this lane's share
    const float c2 = p.scale * kLog2e;

    fetch(0);
    for (int tile = 0; tile < n_tiles; ++tile) {
        __syncthreads();
#pragma unroll
        for (int i = 0; i < kFetchK; ++i) {
            const int e = tid + i * 256;
            store_frag<BF16Elem>(Ks + (e / (DKT * 4)) * LPK + (e % (DKT * 4)) * 8, rk[i]);
        }
#pragma unroll
        for (int i = 0; i < kFetchV; ++i) {
            // keys 8c .. 8c + 7 of a row: two groups of four, each at (group of four in its 16) * 8 + (16 in its 32) * 4
            const int e = tid + i * 256, d = e / (kTileKeys / 8), c = (e % (kTileKeys / 8)) * 8;
            const int in32 = c & 31, at = (c & 32) + ((in32 & 15) / 4) * 8 + (in32 / 16) * 4;
            u32x2_t w[2];
            __builtin_memcpy(w, &rv[i], 16);
            *reinterpret_cast<u32x2_t*>(Vs + d * LPV + at) = w[0];
            *reinterpret_cast<u32x2_t*>(Vs + d * LPV + at + 8) = w[1];
        }
        __syncthreads();
        if (tile + 1 < n_tiles) fetch(tile + 1);
        if (tile * kTileKeys > first_pos + kRowsPerWave - 1) continue;   // no key of this tile for this wave's queries

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
        if (tile * kTileKeys + kTileKeys - 1 > first_pos) {
#pragma unroll
            for (int n = 0; n < 4; ++n)
#pragma unroll
                for (int j = 0; j < 2; ++j)
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        if (tile * kTileKeys + n * 16 + lq * 4 + r > first_pos + j * 16 + l16) s[n][j][r] = -INFINITY;
        }
        typename M::frag fp[2][2];   // [32-key step][query tile]
        float alpha[2];
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            float mx = -INFINITY;
#pragma unroll
            for (int n = 0; n < 4; ++n)
#pragma unroll
                for (int r = 0; r < 4; ++r) mx = fmaxf(mx, s[n][j][r]);
            mx = fmaxf(mx, __shfl_xor(mx, 16));
            mx = fmaxf(mx, __shfl_xor(mx, 32));
            // the scale may be negative or zero only in a configuration error: scores are ordered by s * scale, scale > 0
            const float mn = fmaxf(m[j], mx * c2);
            const float base = mn == -INFINITY ? 0.0f : mn;
            alpha[j] = __builtin_amdgcn_exp2f(m[j] - base);
            m[j] = mn;
            float sum = 0.0f;
#pragma unroll
            for (int n = 0; n < 4; ++n)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float e = __builtin_amdgcn_exp2f(fmaf(s[n][j][r], c2, -base));
                    sum += e;
                    fp[n >> 1][j][(n & 1) * 4 + r] = static_cast<__bf16>(e);
                }
            l[j] = l[j] * alpha[j] + sum;
        }
        if (!__all(alpha[0] == 1.0f && alpha[1] == 1.0f)) {
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
                const typename M::frag fv = M::load(Vs + (d * 16 + l16) * LPV + k * 32 + lq * 8);
                o[d][0] = M::mac(fv, fp[k][0], o[d][0]);
                o[d][1] = M::mac(fv, fp[k][1], o[d][1]);
            }
    }
    const float sk = p.sink[h] * kLog2e;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
        l[j] += __shfl_xor(l[j], 16);
        l[j] += __shfl_xor(l[j], 32);
        const float top = fmaxf(m[j], sk), w = __builtin_amdgcn_exp2f(m[j] - top);
        const float inv = w / (l[j] * w + __builtin_amdgcn_exp2f(sk - top));
        const int t = t0 + wave * kRowsPerWave + j * 16 + l16;
        if (t >= nq) continue;
        uint16_t* out = p.out + ((row0 + static_cast<int64_t>(t)) * p.heads + h) * p.vdim;
#pragma unroll
        for (int d = 0; d < DVT; ++d) {
            const int c = d * 16 + lq * 4;
            if (c < p.vdim) {
                const u32x2_t w2 = {pack_bf16(o[d][j][0] * inv, o[d][j][1] * inv), pack_bf16(o[d][j][2] * inv, o[d][j][3] * inv)};
                *reinterpret_cast<u32x2_t*>(out + c) = w2;
            }
        }
    }
}

template <int DKT, int DVT>
int launch_prompt(const LatentPromptProblem& p, int n_seqs, int max_q, hipStream_t s) {
    const dim3 grid(static_cast<unsigned>(p.heads), static_cast<unsigned>(ceil_div(max_q, kRows)), static_cast<unsigned>(n_seqs));
    launch((latent_prompt_kernel<DKT, DVT>), grid, dim3(256), 0, s, p);
    return launch_status();
}

template <int DVT>
int dispatch_prompt(const LatentPromptProblem& p, int n_seqs, int max_q, hipStream_t s) {
    const int D = p.dim + p.rot;
    if (D <= 64) return launch_prompt<2, DVT>(p, n_seqs, max_q, s);
    if (D <= 96) return launch_prompt<3, DVT>(p, n_seqs, max_q, s);
    if (D <= 128) return launch_prompt<4, DVT>(p, n_seqs, max_q, s);
    if (D <= 192) return launch_prompt<6, DVT>(p, n_seqs, max_q, s);
    return launch_prompt<8, DVT>(p, n_seqs, max_q, s);
}

}  // namespace

// 16-byte pieces of a query, a key and a row of transposed values; registers bound the head sizes
bool latent_prompt_supported(int dim, int rot, int vdim) {
    return dim > 0 && dim % 8 == 0 && rot >= 0 && rot % 8 == 0 && dim + rot <= 256 && vdim > 0 && vdim % 4 == 0 && vdim <= 128;
}

int launch_latent_prompt(const LatentPromptProblem& p, int n_seqs, int max_q, hipStream_t s) {
    return p.vdim <= 64 ? dispatch_prompt<4>(p, n_seqs, max_q, s) : dispatch_prompt<8>(p, n_seqs, max_q, s);
}

}  // namespace em
