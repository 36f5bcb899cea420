// Element types of the hybrid-model kernels: every kernel is instantiated for bfloat16 (the serving type) and
// for float (the same arithmetic with nothing rounded in between).
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#include "../../include/infer_kv.h"

typedef __bf16 bf16x4_t __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4_t __attribute__((ext_vector_type(4)));

constexpr float kLog2e = 1.4426950408889634f;

// N elements at p, widened to float (N = 1, 4 or 8; the pointer is aligned to N elements)
template <int N>
__device__ __forceinline__ void load_elems(const float* p, float (&x)[N]) {
    if constexpr (N % 4 == 0) {
#pragma unroll
        for (int i = 0; i < N / 4; ++i) {
            const f32x4_t v = reinterpret_cast<const f32x4_t*>(p)[i];
#pragma unroll
            for (int e = 0; e < 4; ++e) x[4 * i + e] = v[e];
        }
    } else {
#pragma unroll
        for (int i = 0; i < N; ++i) x[i] = p[i];
    }
}
template <int N>
__device__ __forceinline__ void load_elems(const __bf16* p, float (&x)[N]) {
    if constexpr (N % 4 == 0) {
#pragma unroll
        for (int i = 0; i < N / 4; ++i) {
            const bf16x4_t v = reinterpret_cast<const bf16x4_t*>(p)[i];
#pragma unroll
            for (int e = 0; e < 4; ++e) x[4 * i + e] = (float)v[e];
        }
    } else {
#pragma unroll
        for (int i = 0; i < N; ++i) x[i] = (float)p[i];
    }
}
template <int N>
__device__ __forceinline__ void store_elems(float* p, const float (&x)[N]) {
    if constexpr (N % 4 == 0) {
#pragma unroll
        for (int i = 0; i < N / 4; ++i) {
            f32x4_t v;
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = x[4 * i + e];
            reinterpret_cast<f32x4_t*>(p)[i] = v;
        }
    } else {
#pragma unroll
        for (int i = 0; i < N; ++i) p[i] = x[i];
    }
}
template <int N>
__device__ __forceinline__ void store_elems(__bf16* p, const float (&x)[N]) {
    if constexpr (N % 4 == 0) {
#pragma unroll
        for (int i = 0; i < N / 4; ++i) {
            bf16x4_t v;
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = (__bf16)x[4 * i + e];
            reinterpret_cast<bf16x4_t*>(p)[i] = v;
        }
    } else {
#pragma unroll
        for (int i = 0; i < N; ++i) p[i] = (__bf16)x[i];
    }
}

__device__ __forceinline__ float wave_sum(float x) {
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) x += __shfl_xor(x, m, 64);
    return x;
}

// Sum over a workgroup of WAVES wavefronts; `part` is LDS of WAVES floats that no other reduction in
// flight uses.
template <int WAVES>
__device__ __forceinline__ float block_sum(float x, float* part) {
    x = wave_sum(x);
    if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = x;
    __syncthreads();
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < WAVES; ++i) s += part[i];
    return s;
}

// maximum over the lanes l, l ^ 16, l ^ 32 and l ^ 48, on the vector pipe
__device__ __forceinline__ float max_xor16_32(float x) {
    const unsigned u = __builtin_bit_cast(unsigned, x);
    const auto r = __builtin_amdgcn_permlane16_swap(u, u, false, false);
    const unsigned a0 = r[0], a1 = r[1];
    const float y = fmaxf(__builtin_bit_cast(float, a0), __builtin_bit_cast(float, a1));
    const unsigned w = __builtin_bit_cast(unsigned, y);
    const auto s = __builtin_amdgcn_permlane32_swap(w, w, false, false);
    const unsigned b0 = s[0], b1 = s[1];
    return fmaxf(__builtin_bit_cast(float, b0), __builtin_bit_cast(float, b1));
}

// 1 / (1 + e^-z) by the hardware's exp2 and reciprocal (one unit in the last place each)
__device__ __forceinline__ float sigmoid_f(float z) { return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-kLog2e * z)); }
__device__ __forceinline__ float silu_f(float z) { return z * sigmoid_f(z); }
__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
// 0.5 z (1 + tanh(u)) = z / (1 + exp(-2 u)),  u = sqrt(2 / pi) (z + 0.044715 z^3)
__device__ __forceinline__ float gelu_tanh_f(float z) {
    const float u = 0.7978845608028654f * (z + 0.044715f * z * z * z);
    return z * sigmoid_f(2.0f * u);
}

static inline bool ptr_aligned(const void* p, size_t bytes) { return (reinterpret_cast<uintptr_t>(p) & (bytes - 1)) == 0; }
