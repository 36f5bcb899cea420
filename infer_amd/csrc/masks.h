// Which keys a query sees among those in front of it, and how scores fall with the distance.
#pragma once
#include <stdint.h>

// kind 0: all; 1: those of its chunk, chunks of `size` tokens counted from the sequence's start; 2: itself and the
// size - 1 tokens before it
struct KeyMask {
    int kind = 0, size = 1;
    // the first key that the query at position `pos` sees; it never falls as `pos` grows
    __host__ __device__ __forceinline__ int first(int pos) const {
        if (kind == 0 || pos < 0) return 0;
        if (kind == 1) return pos - pos % size;
        return pos >= size ? pos - size + 1 : 0;
    }
};
static inline bool mask_valid(int kind, int64_t size) { return kind == 0 || ((kind == 1 || kind == 2) && size >= 1 && size <= 0x7fffffff); }

// 2^(-8 (h + 1) / heads)
__device__ __forceinline__ float distance_slope(int h, int heads) { return exp2f(-8.f * (float)(h + 1) / (float)heads); }
