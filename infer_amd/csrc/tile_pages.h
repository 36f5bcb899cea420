// Pages whose tiles of 32 tokens lie in the order in which matrix operands read them, so that keys and values need no staging:
//   keys   [block][kv_head][tile][dim_pad / 32][32 tokens][32 entries]     a k-step of 16 tokens is 1 KiB in a row
//   values [block][kv_head][tile][vdim_pad][32 tokens]                     transposed
// dim_pad and vdim_pad are multiples of 32; entries behind the sizes are zero, tokens behind the last one are anything.
#pragma once
#include <stdint.h>

constexpr int kTileTokens = 32;

// entry d of a token's key, from the tile's start
__host__ __device__ __forceinline__ int tile_key_entry(int token, int d) { return (d >> 5) * 1024 + token * 32 + (d & 31); }
// entry v of a token's value
__host__ __device__ __forceinline__ int tile_value_entry(int token, int v) { return v * 32 + token; }
