// Pages whose tiles of 32 tokens lie in the order in which the lanes of a wavefront read matrix operands (16 x 16 x 32), so that keys and
// values need no staging and every operand is 1 KiB in a row:
//   keys   [block][kv_head][tile][dim_pad / 8][32 tokens][8 entries], of every eight tokens the first four in the tile's first half
//   values [block][kv_head][tile][vdim_pad / 16][4][16 entries][8 tokens]
// dim_pad and vdim_pad are multiples of 32; entries behind the sizes are zero, tokens behind the last one are anything.
#pragma once
#include <stdint.h>

constexpr int kTileTokens = 32;

// Row r of operand x (16 of a tile's keys) is key tile_row_token(r, x), so that the eight results that a lane (g, n) gets of both products,
// rows 4 g + e, are those of the eight consecutive keys 8 g + 4 x + e.
__host__ __device__ __forceinline__ int tile_row_token(int r, int x) { return 8 * (r >> 2) + 4 * x + (r & 3); }

// entry d of a token's key, from the tile's start; the sum of what the token and what the entry contribute
// (and of what is and what is not a multiple of four in the token)
__host__ __device__ __forceinline__ int tile_key_entry(int token, int d) {
    return (d >> 3) * 256 + ((token >> 2 & 1) * 16 + (token >> 3) * 4 + (token & 3)) * 8 + (d & 7);
}
// entry v of a token's value, likewise
__host__ __device__ __forceinline__ int tile_value_entry(int token, int v) { return (v >> 4) * 512 + (token >> 3) * 128 + (v & 15) * 8 + (token & 7); }
