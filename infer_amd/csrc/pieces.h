// Floats as sums of bf16 numbers, so that bf16 matrix instructions can multiply them without giving up float precision.
#pragma once
#include "elem.h"

__device__ __forceinline__ float head(float x) { return __builtin_bit_cast(float, __builtin_bit_cast(uint32_t, x) & 0xffff0000u); }
// the leading halves of two floats, `a` in front
__device__ __forceinline__ uint32_t pack(float a, float b) {
    return __builtin_amdgcn_perm(__builtin_bit_cast(uint32_t, b), __builtin_bit_cast(uint32_t, a), 0x07060302u);
}
__device__ __forceinline__ uint32_t round_pack(float a, float b) {
    typedef __bf16 bf16x2_t __attribute__((ext_vector_type(2)));
    const bf16x2_t r = {(__bf16)a, (__bf16)b};
    return __builtin_bit_cast(uint32_t, r);
}
// N floats as the sum of P bf16 numbers each: the leading 8 bits of the mantissa, the next 8, the last 8 (P = 3: exact;
// P = 2: the second piece rounded)
template <int P, int N>
__device__ __forceinline__ void split(const float (&x)[N], uint32_t (&p)[P][N / 2]) {
#pragma unroll
    for (int i = 0; i < N / 2; ++i) {
        const float a = x[2 * i], b = x[2 * i + 1], ra = a - head(a), rb = b - head(b);
        p[0][i] = pack(a, b);
        if constexpr (P == 2) {
            p[1][i] = round_pack(ra, rb);
        } else {
            p[1][i] = pack(ra, rb);
            p[2][i] = pack(ra - head(ra), rb - head(rb));
        }
    }
}
__device__ __forceinline__ bf16x8_t frag(const uint32_t (&p)[4]) { return __builtin_bit_cast(bf16x8_t, u32x4_t{p[0], p[1], p[2], p[3]}); }
template <int P>
__device__ __forceinline__ void split_frags(const float (&x)[8], bf16x8_t (&f)[P]) {
    uint32_t p[P][4];
    split<P, 8>(x, p);
#pragma unroll
    for (int k = 0; k < P; ++k) f[k] = frag(p[k]);
}

__device__ __forceinline__ void widen(u32x4_t x, float (&y)[8]) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        y[2 * i] = __builtin_bit_cast(float, x[i] << 16);
        y[2 * i + 1] = __builtin_bit_cast(float, x[i] & 0xffff0000u);
    }
}
