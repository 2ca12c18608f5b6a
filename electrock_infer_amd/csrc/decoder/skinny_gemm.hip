// out[T, N] = act(x[T, K] w[N, K]^T) for a decode batch (T <= 64), bf16: a stream over the weights.
//
// A workgroup owns 16 * NT columns of one of `splits` ranges of K; its eight waves share that range out, add their
// results up in LDS, and one pass applies the activation and stores.  A wave reads the weights straight into MFMA operands: per
// 64 elements of k a lane takes 32 consecutive bytes of one row (lane / 16 picks them, so that four lanes cover a
// 128-byte line), for which the k order inside the step is permuted -- the token rows are read in the same order, and a
// sum does not care.  The loads of four such steps are in flight at once.  With splits > 1 the results are float32
// partial sums [splits, T, N] that the next kernel adds up.  GLU: w is [2 N, K], a workgroup makes 16 columns of both
// halves and stores silu(first) * second.
#include "decoder.h"
#include "mma.h"

namespace em {
namespace {

constexpr int kWaves = 8;
constexpr int kStepK = 64;
constexpr int kAhead = 4;

template <int MT, int NT, bool F32OUT, bool GLU = false>
__global__ __launch_bounds__(kWaves * kWave, 2) void skinny_gemm_kernel(const uint16_t* __restrict__ x,
                                                                        const uint16_t* __restrict__ w, void* __restrict__ out,
                                                                        int T, int N, int K, int act) {
    typedef Mma<BF16Elem> M;
    constexpr int kCols = 16 * NT, kTile = 16 * MT * kCols, kOutCols = GLU ? 16 : kCols;
    __shared__ float red[kWaves][kTile];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lq = lane >> 4;
    const int n0 = blockIdx.x * kOutCols;
    const int steps = K / kStepK, splits = gridDim.y, split = blockIdx.y;
    const int g0 = static_cast<int>(static_cast<int64_t>(steps) * split / splits);
    const int g1 = static_cast<int>(static_cast<int64_t>(steps) * (split + 1) / splits);
    const int s0 = g0 + (g1 - g0) * wave / kWaves, s1 = g0 + (g1 - g0) * (wave + 1) / kWaves;

    const uint16_t* wr[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) {
        const int c = n0 + (GLU ? 0 : n * 16) + l16;
        wr[n] = w + (static_cast<int64_t>(c < N ? c : N - 1) + (GLU ? n * static_cast<int64_t>(N) : 0)) * K + lq * 16;   // (columns beyond N are not stored)
    }
    const uint16_t* xr[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        const int t = m * 16 + l16;
        xr[m] = x + static_cast<int64_t>(t < T ? t : T - 1) * K + lq * 16;
    }
    f32x4_t acc[MT][NT];
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int n = 0; n < NT; ++n) acc[m][n] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
    for (int s = s0; s < s1; s += kAhead) {
        typename M::frag fw[kAhead][NT][2];
#pragma unroll
        for (int u = 0; u < kAhead; ++u)
            if (s + u < s1) {
#pragma unroll
                for (int n = 0; n < NT; ++n) {
                    fw[u][n][0] = M::load(wr[n] + (s + u) * kStepK);
                    fw[u][n][1] = M::load(wr[n] + (s + u) * kStepK + 8);
                }
            }
        typename M::frag fx[kAhead][MT][2];
#pragma unroll
        for (int u = 0; u < kAhead; ++u)
            if (s + u < s1) {
#pragma unroll
                for (int m = 0; m < MT; ++m) {
                    fx[u][m][0] = M::load(xr[m] + (s + u) * kStepK);
                    fx[u][m][1] = M::load(xr[m] + (s + u) * kStepK + 8);
                }
            }
#pragma unroll
        for (int u = 0; u < kAhead; ++u)
            if (s + u < s1) {
#pragma unroll
                for (int h = 0; h < 2; ++h)
#pragma unroll
                    for (int m = 0; m < MT; ++m)
#pragma unroll
                        for (int n = 0; n < NT; ++n) acc[m][n] = M::mac(fx[u][m][h], fw[u][n][h], acc[m][n]);
            }
    }
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int n = 0; n < NT; ++n)
#pragma unroll
            for (int r = 0; r < 4; ++r) red[wave][(m * 16 + lq * 4 + r) * kCols + n * 16 + l16] = acc[m][n][r];
    __syncthreads();
    if (GLU) {
        for (int i = tid; i < 16 * MT * 16; i += kWaves * kWave) {
            const int t = i / 16, c = i % 16;
            if (t >= T || n0 + c >= N) continue;
            float g = 0.0f, u = 0.0f;
#pragma unroll
            for (int k = 0; k < kWaves; ++k) {
                g += red[k][t * kCols + c];
                u += red[k][t * kCols + 16 + c];
            }
            static_cast<uint16_t*>(out)[static_cast<int64_t>(t) * N + n0 + c] = f32_to_bf16_bits(silu(g) * u);
        }
        return;
    }
    for (int i = tid; i < kTile; i += kWaves * kWave) {
        const int t = i / kCols, c = n0 + i % kCols;
        if (t >= T || c >= N) continue;
        float v = 0.0f;
#pragma unroll
        for (int k = 0; k < kWaves; ++k) v += red[k][i];
        if (act == 1) {
            v = fmaxf(v, 0.0f);
            v *= v;
        }
        const int64_t at = (static_cast<int64_t>(split) * T + t) * N + c;
        if (F32OUT) static_cast<float*>(out)[at] = v;
        else static_cast<uint16_t*>(out)[at] = f32_to_bf16_bits(v);
    }
}

template <int MT>
int launch_glu(const uint16_t* x, const uint16_t* w, void* out, int T, int N, int K, hipStream_t s) {
    launch((skinny_gemm_kernel<MT, 2, false, true>), dim3(static_cast<unsigned>(ceil_div(N, 16))), dim3(kWaves * kWave), 0, s, x, w, out, T, N, K, 0);
    return launch_status();
}

template <int MT, int NT>
int launch_skinny(const uint16_t* x, const uint16_t* w, void* out, bool f32, int splits, int T, int N, int K, int act, hipStream_t s) {
    const dim3 grid(static_cast<unsigned>(ceil_div(N, 16 * NT)), static_cast<unsigned>(splits)), block(kWaves * kWave);
    if (f32) launch((skinny_gemm_kernel<MT, NT, true>), grid, block, 0, s, x, w, out, T, N, K, act);
    else launch((skinny_gemm_kernel<MT, NT, false>), grid, block, 0, s, x, w, out, T, N, K, act);
    return launch_status();
}

int cols_per_group(int T, int N) { return T <= 16 && N <= 8192 ? 16 : 32; }

}  // namespace

// The range where this beats the library's product, which is slower to get going: up to 16 tokens unless the weights are
// large, up to 64 tokens for small ones (us, this / library; 6144 x 2048: T = 1 8.6 / 12.4, T = 16 11.1 / 12.3, T = 32
// 11.0 / 12.5, T = 64 15.3 / 13.0; 2048 x 2048, T = 64: 6.3 / 8.8; 12288 x 4096: T = 1 24.9 / 26.6, T = 16 29.7 / 25.7).
bool skinny_supported(int64_t T, int N, int K) {
    if (T <= 0 || N <= 0 || K <= 0 || K % kStepK != 0) return false;
    const int64_t weights = static_cast<int64_t>(N) * K;
    return T <= 4 || (T <= 16 && weights <= (int64_t{1} << 25)) || (T <= 32 && weights <= (int64_t{1} << 24)) ||
           (T <= 64 && weights <= (int64_t{1} << 22));
}

// Ranges of K for results that may stay partial sums: enough workgroups for the chip, a step of k for every wave.
int skinny_splits(int T, int N, int K) {
    const int groups = static_cast<int>(ceil_div(N, cols_per_group(T, N)));
    const int want = static_cast<int>(ceil_div(384, groups)), most = K / (kStepK * kWaves);
    const int s = want < most ? want : most;
    return s < 1 ? 1 : s > 8 ? 8 : s;
}

int launch_skinny_gemm(const void* x, const void* w, void* out, bool f32, int splits, int T, int N, int K, int act, hipStream_t s) {
    const uint16_t* xp = static_cast<const uint16_t*>(x);
    const uint16_t* wp = static_cast<const uint16_t*>(w);
    if (act == 2) return T <= 16 ? launch_glu<1>(xp, wp, out, T, N, K, s) : T <= 32 ? launch_glu<2>(xp, wp, out, T, N, K, s) : launch_glu<4>(xp, wp, out, T, N, K, s);
    if (cols_per_group(T, N) == 16) return launch_skinny<1, 1>(xp, wp, out, f32, splits, T, N, K, act, s);
    if (T <= 16) return launch_skinny<1, 2>(xp, wp, out, f32, splits, T, N, K, act, s);
    if (T <= 32) return launch_skinny<2, 2>(xp, wp, out, f32, splits, T, N, K, act, s);
    return launch_skinny<4, 2>(xp, wp, out, f32, splits, T, N, K, act, s);
}

}  // namespace em
