// 16 x 16 x 32 matrix step for bf16 and for float32 operands with one register layout, and the loads that feed it.
//
// A wave multiplies A [16 x 32] by B [32 x 16]: lane l holds the eight values k = (l / 16) * 8 + 0..7 of row l % 16 of A
// and of column l % 16 of B; of the result it holds column l % 16 of the rows (l / 16) * 4 + 0..3.  bf16 is one
// 16x16x32 MFMA.  float32 is eight 16x16x4 MFMAs, the i-th of which takes value i of every lane (the sum over k does
// not care which k an instruction sees as long as A and B agree), so kernels written on these fragments serve both.
#pragma once
#include "../common.h"

namespace em {

typedef float f32x8_t __attribute__((ext_vector_type(8)));

template <typename Elem> struct Mma;

template <> struct Mma<BF16Elem> {
    typedef bf16x8_t frag;
    static __device__ __forceinline__ frag zero() {
        frag f;
#pragma unroll
        for (int i = 0; i < 8; ++i) f[i] = static_cast<__bf16>(0.0f);
        return f;
    }
    static __device__ __forceinline__ frag load(const uint16_t* p) {  // 16-byte aligned
        frag f;
        const u32x4_t w = *reinterpret_cast<const u32x4_t*>(p);
        __builtin_memcpy(&f, &w, 16);
        return f;
    }
    static __device__ __forceinline__ void set(frag& f, int i, uint16_t bits) {
        __bf16 b;
        __builtin_memcpy(&b, &bits, 2);
        f[i] = b;
    }
    static __device__ __forceinline__ f32x4_t mac(frag a, frag b, f32x4_t c) {
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
    }
};

template <> struct Mma<F32Elem> {
    typedef f32x8_t frag;
    static __device__ __forceinline__ frag zero() {
        frag f;
#pragma unroll
        for (int i = 0; i < 8; ++i) f[i] = 0.0f;
        return f;
    }
    static __device__ __forceinline__ frag load(const float* p) {
        frag f;
        const f32x4_t lo = *reinterpret_cast<const f32x4_t*>(p), hi = *reinterpret_cast<const f32x4_t*>(p + 4);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            f[i] = lo[i];
            f[i + 4] = hi[i];
        }
        return f;
    }
    static __device__ __forceinline__ void set(frag& f, int i, float v) { f[i] = v; }
    static __device__ __forceinline__ f32x4_t mac(frag a, frag b, f32x4_t c) {
#pragma unroll
        for (int i = 0; i < 8; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
        return c;
    }
};

// Eight consecutive elements of which the first `valid` exist (the rest read as zero).  `vec`: the caller knows that
// the address is aligned to the eight elements' size.
template <typename Elem>
__device__ __forceinline__ typename Mma<Elem>::frag load_frag(const typename Elem::storage* p, int valid, bool vec) {
    if (vec && valid >= 8) return Mma<Elem>::load(p);
    typename Mma<Elem>::frag f = Mma<Elem>::zero();
#pragma unroll
    for (int i = 0; i < 8; ++i)
        if (i < valid) Mma<Elem>::set(f, i, p[i]);
    return f;
}

// Eight elements into LDS or global memory, aligned.
template <typename Elem>
__device__ __forceinline__ void store_frag(typename Elem::storage* p, typename Mma<Elem>::frag f) {
    constexpr int kWords = sizeof(typename Elem::storage) * 8 / 16;
    u32x4_t w[kWords];
    __builtin_memcpy(w, &f, sizeof(w));
#pragma unroll
    for (int i = 0; i < kWords; ++i) reinterpret_cast<u32x4_t*>(p)[i] = w[i];
}

}  // namespace em
