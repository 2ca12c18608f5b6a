// Row kernels of a decoder whose residual stream is float32: embedding, post-norm residual update fused with the next
// layer's pre-norm, squared ReLU, gated SiLU, and the gated norm of a mixer's output.
#include "decoder.h"

namespace em {
namespace {

constexpr int kRowMaxPerThread = 32;  // floats of a row that one thread keeps in registers

// Sum over the workgroup, the same value and the same order in every thread.  `scratch`: one float per wave.
template <int THREADS>
__device__ __forceinline__ float block_sum(float v, float* scratch) {
#pragma unroll
    for (int off = kWave / 2; off > 0; off >>= 1) v += __shfl_xor(v, off);
    __syncthreads();  // readers of an earlier sum are done
    if (lane_id() == 0) scratch[threadIdx.x / kWave] = v;
    __syncthreads();
    float total = 0.0f;
#pragma unroll
    for (int w = 0; w < THREADS / kWave; ++w) total += scratch[w];
    return total;
}

template <typename Elem, int VEC>
struct RowIo {
    static __device__ __forceinline__ void load(const typename Elem::storage* p, float (&v)[VEC]) {
        typename Elem::storage t[VEC];
        __builtin_memcpy(t, __builtin_assume_aligned(p, VEC * sizeof(t[0])), sizeof(t));
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] = Elem::load(t[j]);
    }
    static __device__ __forceinline__ void store(typename Elem::storage* p, const float (&v)[VEC]) {
        typename Elem::storage t[VEC];
#pragma unroll
        for (int j = 0; j < VEC; ++j) t[j] = Elem::store(v[j]);
        __builtin_memcpy(__builtin_assume_aligned(p, VEC * sizeof(t[0])), t, sizeof(t));
    }
};

// x = table[token] * scale in float32; copied, rounded to the compute type, to up to two strided destinations.
template <typename Elem, int VEC>
__global__ __launch_bounds__(256) void embed_kernel(const int32_t* __restrict__ tokens,
                                                    const typename Elem::storage* __restrict__ table, float scale,
                                                    float* __restrict__ x, typename Elem::storage* __restrict__ copy,
                                                    int64_t copy_stride, int W) {
    const int64_t t = blockIdx.x;
    const typename Elem::storage* src = table + static_cast<int64_t>(tokens[t]) * W;
    for (int c = threadIdx.x * VEC; c < W; c += 256 * VEC) {
        float v[VEC];
        RowIo<Elem, VEC>::load(src + c, v);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] *= scale;
        RowIo<F32Elem, VEC>::store(x + t * W + c, v);
        if (copy != nullptr) RowIo<Elem, VEC>::store(copy + t * copy_stride + c, v);
    }
}

// One workgroup per row.
// y may be given as float32 partial sums [y_parts, T, W].
//   UPDATE 0: x stays          UPDATE 1: x += y / rms(y) * post_w          UPDATE 2: x = y + post_w
//   then, when out != null: out = next_w ? x / rms(x) * next_w : x, rounded to the compute type
template <typename Elem, typename YElem, int UPDATE, int VEC, int THREADS>
__global__ __launch_bounds__(THREADS) void residual_norm_kernel(
    float* __restrict__ x, const typename YElem::storage* __restrict__ y, int y_parts, const float* __restrict__ post_w,
    const float* __restrict__ next_w, typename Elem::storage* __restrict__ out, int64_t out_stride, int W, float eps) {
    __shared__ float scratch[THREADS / kWave];
    constexpr int N = kRowMaxPerThread / VEC;
    const int64_t row = blockIdx.x;
    float* xr = x + row * W;
    float v[N][VEC];
    if (UPDATE != 0) {
        const typename YElem::storage* yr = y + row * W;
        float sum = 0.0f;
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const int c = (threadIdx.x + i * THREADS) * VEC;
            if (c < W) {
                RowIo<YElem, VEC>::load(yr + c, v[i]);
                for (int p = 1; p < y_parts; ++p) {
                    float more[VEC];
                    RowIo<YElem, VEC>::load(yr + static_cast<int64_t>(p) * gridDim.x * W + c, more);
#pragma unroll
                    for (int j = 0; j < VEC; ++j) v[i][j] += more[j];
                }
#pragma unroll
                for (int j = 0; j < VEC; ++j) sum = fmaf(v[i][j], v[i][j], sum);
            }
        }
        float rstd = 0.0f;
        if (UPDATE == 1) rstd = 1.0f / sqrtf(block_sum<THREADS>(sum, scratch) / static_cast<float>(W) + eps);
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const int c = (threadIdx.x + i * THREADS) * VEC;
            if (c < W) {
                float pw[VEC];
                if (UPDATE == 1) {
                    float xv[VEC];
                    RowIo<F32Elem, VEC>::load(post_w + c, pw);
                    RowIo<F32Elem, VEC>::load(xr + c, xv);
#pragma unroll
                    for (int j = 0; j < VEC; ++j) v[i][j] = xv[j] + v[i][j] * rstd * pw[j];
                } else if (post_w != nullptr) {
                    RowIo<F32Elem, VEC>::load(post_w + c, pw);
#pragma unroll
                    for (int j = 0; j < VEC; ++j) v[i][j] += pw[j];
                }
                RowIo<F32Elem, VEC>::store(xr + c, v[i]);
            }
        }
    } else {
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const int c = (threadIdx.x + i * THREADS) * VEC;
            if (c < W) RowIo<F32Elem, VEC>::load(xr + c, v[i]);
        }
    }
    if (out == nullptr) return;
    float rstd = 1.0f;
    if (next_w != nullptr) {
        float sum = 0.0f;
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const int c = (threadIdx.x + i * THREADS) * VEC;
            if (c < W) {
#pragma unroll
                for (int j = 0; j < VEC; ++j) sum = fmaf(v[i][j], v[i][j], sum);
            }
        }
        rstd = 1.0f / sqrtf(block_sum<THREADS>(sum, scratch) / static_cast<float>(W) + eps);
    }
#pragma unroll
    for (int i = 0; i < N; ++i) {
        const int c = (threadIdx.x + i * THREADS) * VEC;
        if (c < W) {
            float o[VEC];
            if (next_w != nullptr) {
                float nw[VEC];
                RowIo<F32Elem, VEC>::load(next_w + c, nw);
#pragma unroll
                for (int j = 0; j < VEC; ++j) o[j] = v[i][j] * rstd * nw[j];
            } else {
#pragma unroll
                for (int j = 0; j < VEC; ++j) o[j] = v[i][j];
            }
            RowIo<Elem, VEC>::store(out + row * out_stride + c, o);
        }
    }
}

// u = relu(u)^2 in place
template <typename Elem, int VEC>
__global__ __launch_bounds__(256) void relu_squared_kernel(typename Elem::storage* __restrict__ u, int64_t n) {
    const int64_t i = (static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x) * VEC;
    if (i >= n) return;
    float v[VEC];
    RowIo<Elem, VEC>::load(u + i, v);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
        const float r = fmaxf(v[j], 0.0f);
        v[j] = r * r;
    }
    RowIo<Elem, VEC>::store(u + i, v);
}

// out [T, ff] = silu(u[:, :ff]) * u[:, ff:]
template <typename Elem, int VEC>
__global__ __launch_bounds__(256) void silu_gate_kernel(const typename Elem::storage* __restrict__ u, typename Elem::storage* __restrict__ out,
                                                        int64_t n, int ff) {
    const int64_t i = (static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x) * VEC;
    if (i >= n) return;
    const int64_t row = i / ff, c = i - row * ff;
    float g[VEC], v[VEC];
    RowIo<Elem, VEC>::load(u + row * 2 * ff + c, g);
    RowIo<Elem, VEC>::load(u + row * 2 * ff + ff + c, v);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] *= silu(g[j]);
    RowIo<Elem, VEC>::store(out + i, v);
}

// y = y silu(z), normed in equal parts of `size` elements, times w, in place: one workgroup per (row, part)
template <typename Elem, int VEC, int THREADS>
__global__ __launch_bounds__(THREADS) void gated_norm_kernel(typename Elem::storage* __restrict__ y, const typename Elem::storage* __restrict__ z,
                                                             int64_t z_stride, const float* __restrict__ w, int size, float eps) {
    __shared__ float scratch[THREADS / kWave];
    constexpr int N = kRowMaxPerThread / VEC;
    const int64_t row = blockIdx.x;
    const int c0 = blockIdx.y * size;
    typename Elem::storage* yr = y + (row * gridDim.y + blockIdx.y) * size;
    const typename Elem::storage* zr = z + row * z_stride + c0;
    float v[N][VEC], sum = 0.0f;
#pragma unroll
    for (int i = 0; i < N; ++i) {
        const int c = (threadIdx.x + i * THREADS) * VEC;
        if (c < size) {
            float g[VEC];
            RowIo<Elem, VEC>::load(yr + c, v[i]);
            RowIo<Elem, VEC>::load(zr + c, g);
#pragma unroll
            for (int j = 0; j < VEC; ++j) {
                v[i][j] *= silu(g[j]);
                sum = fmaf(v[i][j], v[i][j], sum);
            }
        }
    }
    const float rstd = 1.0f / sqrtf(block_sum<THREADS>(sum, scratch) / static_cast<float>(size) + eps);
#pragma unroll
    for (int i = 0; i < N; ++i) {
        const int c = (threadIdx.x + i * THREADS) * VEC;
        if (c < size) {
            float wv[VEC];
            RowIo<F32Elem, VEC>::load(w + c0 + c, wv);
#pragma unroll
            for (int j = 0; j < VEC; ++j) v[i][j] *= rstd * wv[j];
            RowIo<Elem, VEC>::store(yr + c, v[i]);
        }
    }
}

template <typename Elem, int VEC>
int launch_gated(void* y, const void* z, int64_t z_stride, const float* w, int64_t T, int parts, int size, float eps, hipStream_t s) {
    typedef typename Elem::storage S;
    const dim3 grid(static_cast<unsigned>(T), static_cast<unsigned>(parts));
    if (size <= 64 * kRowMaxPerThread / 4)
        launch((gated_norm_kernel<Elem, VEC, 64>), grid, dim3(64), 0, s, static_cast<S*>(y), static_cast<const S*>(z), z_stride, w, size, eps);
    else if (size <= 256 * kRowMaxPerThread)
        launch((gated_norm_kernel<Elem, VEC, 256>), grid, dim3(256), 0, s, static_cast<S*>(y), static_cast<const S*>(z), z_stride, w, size, eps);
    else
        launch((gated_norm_kernel<Elem, VEC, 1024>), grid, dim3(1024), 0, s, static_cast<S*>(y), static_cast<const S*>(z), z_stride, w, size, eps);
    return launch_status();
}

template <typename Elem, typename YElem, int UPDATE, int VEC>
int launch_residual(float* x, const void* y, int y_parts, const float* post_w, const float* next_w, void* out, int64_t out_stride,
                    int64_t T, int W, float eps, hipStream_t s) {
    typedef typename Elem::storage S;
    typedef typename YElem::storage YS;
    const dim3 grid(static_cast<unsigned>(T));
    if (W <= 256 * kRowMaxPerThread)
        launch((residual_norm_kernel<Elem, YElem, UPDATE, VEC, 256>), grid, dim3(256), 0, s, x,
               static_cast<const YS*>(y), y_parts, post_w, next_w, static_cast<S*>(out), out_stride, W, eps);
    else
        launch((residual_norm_kernel<Elem, YElem, UPDATE, VEC, 1024>), grid, dim3(1024), 0, s, x,
               static_cast<const YS*>(y), y_parts, post_w, next_w, static_cast<S*>(out), out_stride, W, eps);
    return launch_status();
}

template <typename Elem, typename YElem, int VEC>
int dispatch_residual(int update, float* x, const void* y, int y_parts, const float* post_w, const float* next_w, void* out,
                      int64_t out_stride, int64_t T, int W, float eps, hipStream_t s) {
    if (update == 0) return launch_residual<Elem, YElem, 0, VEC>(x, y, y_parts, post_w, next_w, out, out_stride, T, W, eps, s);
    if (update == 1) return launch_residual<Elem, YElem, 1, VEC>(x, y, y_parts, post_w, next_w, out, out_stride, T, W, eps, s);
    return launch_residual<Elem, YElem, 2, VEC>(x, y, y_parts, post_w, next_w, out, out_stride, T, W, eps, s);
}

}  // namespace

bool row_width_ok(int W) { return W > 0 && W <= 1024 * kRowMaxPerThread; }

int launch_embed(const int32_t* tokens, const void* table, float scale, float* x, void* copy, int64_t copy_stride,
                 int64_t T, int W, int dtype, hipStream_t s) {
    const dim3 grid(static_cast<unsigned>(T));
    const bool vec = W % 4 == 0 && copy_stride % 4 == 0;
    if (dtype == EM_DTYPE_BF16) {
        const uint16_t* e = static_cast<const uint16_t*>(table);
        uint16_t* c = static_cast<uint16_t*>(copy);
        if (vec) launch((embed_kernel<BF16Elem, 4>), grid, dim3(256), 0, s, tokens, e, scale, x, c, copy_stride, W);
        else launch((embed_kernel<BF16Elem, 1>), grid, dim3(256), 0, s, tokens, e, scale, x, c, copy_stride, W);
    } else {
        const float* e = static_cast<const float*>(table);
        float* c = static_cast<float*>(copy);
        if (vec) launch((embed_kernel<F32Elem, 4>), grid, dim3(256), 0, s, tokens, e, scale, x, c, copy_stride, W);
        else launch((embed_kernel<F32Elem, 1>), grid, dim3(256), 0, s, tokens, e, scale, x, c, copy_stride, W);
    }
    return launch_status();
}

int launch_residual_norm(int update, float* x, const void* y, int y_dtype, int y_parts, const float* post_w, const float* next_w,
                         void* out, int64_t out_stride, int64_t T, int W, float eps, int dtype, hipStream_t s) {
    const bool vec = W % 4 == 0 && out_stride % 4 == 0;
#define EM_RESIDUAL(E, Y)                                                                                        \
    return vec ? dispatch_residual<E, Y, 4>(update, x, y, y_parts, post_w, next_w, out, out_stride, T, W, eps, s)         \
               : dispatch_residual<E, Y, 1>(update, x, y, y_parts, post_w, next_w, out, out_stride, T, W, eps, s)
    if (dtype == EM_DTYPE_F32) { EM_RESIDUAL(F32Elem, F32Elem); }
    if (y_dtype == EM_DTYPE_F32) { EM_RESIDUAL(BF16Elem, F32Elem); }
    EM_RESIDUAL(BF16Elem, BF16Elem);
#undef EM_RESIDUAL
}

int launch_relu_squared(void* u, int64_t n, int dtype, hipStream_t s) {
    const int vec = n % 8 == 0 ? 8 : 1;
    const dim3 grid(static_cast<unsigned>(ceil_div(ceil_div(n, vec), 256)));
    if (dtype == EM_DTYPE_BF16) {
        if (vec == 8) launch((relu_squared_kernel<BF16Elem, 8>), grid, dim3(256), 0, s, static_cast<uint16_t*>(u), n);
        else launch((relu_squared_kernel<BF16Elem, 1>), grid, dim3(256), 0, s, static_cast<uint16_t*>(u), n);
    } else {
        if (vec == 8) launch((relu_squared_kernel<F32Elem, 8>), grid, dim3(256), 0, s, static_cast<float*>(u), n);
        else launch((relu_squared_kernel<F32Elem, 1>), grid, dim3(256), 0, s, static_cast<float*>(u), n);
    }
    return launch_status();
}

int launch_silu_gate(const void* u, void* out, int64_t T, int ff, int dtype, hipStream_t s) {
    const int64_t n = T * ff;
    const int vec = ff % 8 == 0 ? 8 : 1;
    const dim3 grid(static_cast<unsigned>(ceil_div(ceil_div(n, vec), 256)));
    if (dtype == EM_DTYPE_BF16) {
        if (vec == 8) launch((silu_gate_kernel<BF16Elem, 8>), grid, dim3(256), 0, s, static_cast<const uint16_t*>(u), static_cast<uint16_t*>(out), n, ff);
        else launch((silu_gate_kernel<BF16Elem, 1>), grid, dim3(256), 0, s, static_cast<const uint16_t*>(u), static_cast<uint16_t*>(out), n, ff);
    } else {
        if (vec == 8) launch((silu_gate_kernel<F32Elem, 8>), grid, dim3(256), 0, s, static_cast<const float*>(u), static_cast<float*>(out), n, ff);
        else launch((silu_gate_kernel<F32Elem, 1>), grid, dim3(256), 0, s, static_cast<const float*>(u), static_cast<float*>(out), n, ff);
    }
    return launch_status();
}

int launch_gated_norm(void* y, const void* z, int64_t z_stride, const float* w, int64_t T, int parts, int size, float eps, int dtype,
                      hipStream_t s) {
    const bool vec = size % 4 == 0 && z_stride % 4 == 0;
    if (dtype == EM_DTYPE_BF16)
        return vec ? launch_gated<BF16Elem, 4>(y, z, z_stride, w, T, parts, size, eps, s)
                   : launch_gated<BF16Elem, 1>(y, z, z_stride, w, T, parts, size, eps, s);
    return vec ? launch_gated<F32Elem, 4>(y, z, z_stride, w, T, parts, size, eps, s)
               : launch_gated<F32Elem, 1>(y, z, z_stride, w, T, parts, size, eps, s);
}

}  // namespace em
