// Mixture of experts, for gfx950 (MI355X).
//
//   moe_logits_kernel / moe_route_*   router logits in float32, softmax, the choice of experts inside the best groups, weights, and
//                                     every choice's rank among the choices of its expert
//   moe_scatter_kernel    rows sorted by expert: place of every choice, token and expert of every place, row tiles
//   moe_block_kernel      products of many rows per expert: 256 rows x 256 columns per workgroup, straight from memory to LDS
//   moe_tile_kernel       products of large row tiles: 128 rows x 128 columns per workgroup, through registers to LDS
//   moe_row_kernel        products of 16-row tiles (decode): the weights stream past the rows, k split over wavefronts
//   moe_any_kernel        any size and element type
//
// The first product takes gate and up columns side by side and stores act = silu(gate) * up, the second stores one row per
// place; the weighted sum of a token's rows is part of the next residual step (pre_norm.hip).  A choice beyond the experts is
// the identity: place -1, no row.
#include "elem.h"

namespace {

constexpr int kThreads = 256;
constexpr int kMaxExperts = 1024;

template <class T>
struct RouteArgs {
    const T* h; int64_t h_stride;
    const T* router;                       // [all][width]
    const float* correction;               // [all] or nullptr
    int width, all, experts, top, groups, keep;
    float scale;
    int32_t* ids; float* weights; int32_t* ranks;      // [n][top]
    int32_t* counts;                       // [experts], zero before
    int n;
};

// The choices of one token by one wavefront; `z` are its logits in LDS.  Ties go to the lower index.
template <int NE, class T>
__device__ __forceinline__ void choose(const RouteArgs<T>& a, const float* z, int64_t token, int* hist, int* rank_out) {
    const int lane = threadIdx.x & 63, size = a.all / a.groups;
    float s[NE], c[NE];
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
        const int e = lane + 64 * i;
        s[i] = e < a.all ? z[e] : -INFINITY;
        mx = fmaxf(mx, s[i]);
    }
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) mx = fmaxf(mx, __shfl_xor(mx, m, 64));
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
        s[i] = expf(s[i] - mx);
        sum += s[i];
    }
    sum = wave_sum(sum);
    unsigned open = 0;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
        const int e = lane + 64 * i;
        s[i] /= sum;
        c[i] = e < a.all ? s[i] + (a.correction ? a.correction[e] : 0.f) : -INFINITY;
        if (e < a.all && a.keep >= a.groups) open |= 1u << i;
    }
    // the largest of the entries whose bit in `of` is set; -1: none
    auto best = [&](unsigned of) {
        float v = -INFINITY;
        int at = 0x7fffffff;
#pragma unroll
        for (int i = 0; i < NE; ++i)
            if ((of >> i & 1u) && (at == 0x7fffffff || c[i] > v)) { v = c[i]; at = lane + 64 * i; }
#pragma unroll
        for (int m = 32; m >= 1; m >>= 1) {
            const float ov = __shfl_xor(v, m, 64);
            const int oat = __shfl_xor(at, m, 64);
            if (oat != 0x7fffffff && (at == 0x7fffffff || ov > v || (ov == v && oat < at))) { v = ov; at = oat; }
        }
        return at == 0x7fffffff ? -1 : at;
    };
    if (a.keep < a.groups) {               // groups in the order of their largest entry
        unsigned valid = 0;
#pragma unroll
        for (int i = 0; i < NE; ++i)
            if (lane + 64 * i < a.all) valid |= 1u << i;
        for (int k = 0; k < a.keep; ++k) {
            const int at = best(valid & ~open), grp = at < 0 ? -1 : at / size;
#pragma unroll
            for (int i = 0; i < NE; ++i)
                if (lane + 64 * i < a.all && (lane + 64 * i) / size == grp) open |= 1u << i;
        }
    }
    int id = 0;
    float w = 0.f;
    for (int k = 0; k < a.top; ++k) {
        const int at = best(open);
        float v = 0.f;
#pragma unroll
        for (int i = 0; i < NE; ++i)
            if (at == lane + 64 * i) { v = s[i]; open &= ~(1u << i); }
        v = at < 0 ? 0.f : __shfl(v, at & 63, 64);
        if (lane == k) { id = at < 0 ? a.all - 1 : at; w = v * a.scale; }
    }
    if (lane < a.top) {
        a.ids[token * a.top + lane] = id;
        a.weights[token * a.top + lane] = w;
        rank_out[lane] = id < a.experts ? atomicAdd(&hist[id], 1) : 0;
    }
}

// behind the choices of a workgroup's tokens: their ranks among all choices of their experts
template <class T>
__device__ __forceinline__ void finish_ranks(const RouteArgs<T>& a, int64_t token0, int tokens, int* hist, const int* ranks) {
    const int threads = blockDim.x;
    __syncthreads();
    for (int e = threadIdx.x; e < a.experts; e += threads) {
        const int c = hist[e];
        hist[e] = c ? atomicAdd(&a.counts[e], c) : 0;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < tokens * a.top; i += threads) {
        const int64_t at = token0 * a.top + i;
        const int id = a.ids[at];
        a.ranks[at] = id < a.experts ? hist[id] + ranks[i] : 0;
    }
}

// ET tiles of 16 experts, U tiles of 16 tokens per workgroup; wavefront w of W takes the k-steps w, w + W, ...  Few tokens: one tile
// and many wavefronts, so that the chain of requests is short; many tokens: two tiles, so that the router is read half as often.
template <int ET, int U, int W>
__global__ void __launch_bounds__(64 * W) moe_route_tile_kernel(RouteArgs<__bf16> a) {
    constexpr int kRow = 16 * ET + 1, kAhead = U + ET <= 3 ? 8 : U + ET <= 6 ? 4 : 2;
    __shared__ float z[16 * U * kRow];
    __shared__ int hist[kMaxExperts], ranks[16 * U * 64];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, n = lane & 15;
    const int64_t token0 = (int64_t)blockIdx.x * (16 * U);
    for (int e = tid; e < a.experts; e += 64 * W) hist[e] = 0;
    f32x4_t acc[U][ET];
    const __bf16* hr[U];
    const __bf16* rr[ET];
#pragma unroll
    for (int u = 0; u < U; ++u) {
        const int64_t t = token0 + 16 * u + n;
        hr[u] = a.h + (t < a.n ? t : a.n - 1) * a.h_stride + 8 * g;
#pragma unroll
        for (int i = 0; i < ET; ++i) acc[u][i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int i = 0; i < ET; ++i) rr[i] = a.router + (int64_t)(16 * i + n < a.all ? 16 * i + n : a.all - 1) * a.width + 8 * g;
#pragma unroll kAhead
    for (int k = 32 * wave; k < a.width; k += 32 * W) {
        bf16x8_t x[U];
#pragma unroll
        for (int u = 0; u < U; ++u) x[u] = *reinterpret_cast<const bf16x8_t*>(hr[u] + k);
#pragma unroll
        for (int i = 0; i < ET; ++i) {
            const bf16x8_t w = *reinterpret_cast<const bf16x8_t*>(rr[i] + k);
#pragma unroll
            for (int u = 0; u < U; ++u) acc[u][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w, x[u], acc[u][i], 0, 0, 0);
        }
    }
    for (int w = 0; w < W; ++w) {
        if (wave == w)
#pragma unroll
            for (int u = 0; u < U; ++u)
#pragma unroll
                for (int i = 0; i < ET; ++i)
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        float* p = z + (16 * u + n) * kRow + 16 * i + 4 * g + e;
                        *p = w == 0 ? acc[u][i][e] : *p + acc[u][i][e];
                    }
        __syncthreads();
    }
    const int tokens = token0 + 16 * U < a.n ? 16 * U : (int)(a.n - token0);
    for (int t = wave; t < tokens; t += W) choose<(ET + 3) / 4>(a, z + t * kRow, token0 + t, hist, ranks + t * a.top);
    finish_ranks(a, token0, tokens, hist, ranks);
}

template <int ET>
void launch_route(const RouteArgs<__bf16>& a, hipStream_t st) {
    if (a.n <= 2048) hipLaunchKernelGGL((moe_route_tile_kernel<ET, 1, 16>), dim3((unsigned)((a.n + 15) / 16)), dim3(1024), 0, st, a);
    else hipLaunchKernelGGL((moe_route_tile_kernel<ET, 2, 4>), dim3((unsigned)((a.n + 31) / 32)), dim3(256), 0, st, a);
}

// any size: one token per wavefront, four per workgroup
template <class T>
__global__ void __launch_bounds__(kThreads) moe_route_any_kernel(RouteArgs<T> a) {
    __shared__ float z[4][kMaxExperts];
    __shared__ int hist[kMaxExperts], ranks[4 * 64];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int64_t token0 = (int64_t)blockIdx.x * 4;
    const int tokens = token0 + 4 < a.n ? 4 : (int)(a.n - token0);
    for (int e = tid; e < a.experts; e += kThreads) hist[e] = 0;
    if (wave < tokens) {
        const T* h = a.h + (token0 + wave) * a.h_stride;
        for (int e = 0; e < a.all; ++e) {
            const T* r = a.router + (int64_t)e * a.width;
            float s = 0.f;
            for (int c = lane; c < a.width; c += 64) s += (float)h[c] * (float)r[c];
            s = wave_sum(s);
            if (lane == 0) z[wave][e] = s;
        }
    }
    __syncthreads();
    if (wave < tokens) choose<kMaxExperts / 64>(a, z[wave], token0 + wave, hist, ranks + wave * a.top);
    finish_ranks(a, token0, tokens, hist, ranks);
}

struct ScatterArgs {
    const int32_t* ids; const int32_t* ranks; const int32_t* counts;
    int experts, top, tile_rows, max_tiles;
    int64_t choices;
    int32_t* places;                       // [choices]
    int32_t* row_token; int32_t* row_expert;           // [place]
    int32_t* offsets;                      // [experts + 1]
    int32_t* tiles;                        // [max_tiles][2]: expert (-1: none), first row inside the expert
};

// exclusive prefix sum over the workgroup
__device__ __forceinline__ int block_scan(int x, int* part) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    int s = x;
#pragma unroll
    for (int m = 1; m < 64; m <<= 1) {
        const int up = __shfl_up(s, m, 64);
        if (lane >= m) s += up;
    }
    if (lane == 63) part[wave] = s;
    __syncthreads();
    int before = 0;
    for (int i = 0; i < wave; ++i) before += part[i];
    return before + s - x;
}

__global__ void __launch_bounds__(kThreads) moe_scatter_kernel(ScatterArgs a) {
    __shared__ int off[kMaxExperts + 4], part[2][4];
    const int tid = threadIdx.x;
    constexpr int kPer = kMaxExperts / kThreads;
    int cnt[kPer], rows = 0, tiles = 0;
#pragma unroll
    for (int i = 0; i < kPer; ++i) {
        const int e = kPer * tid + i;
        cnt[i] = e < a.experts ? a.counts[e] : 0;
        rows += cnt[i];
        tiles += (cnt[i] + a.tile_rows - 1) / a.tile_rows;
    }
    int row0 = block_scan(rows, part[0]), tile0 = block_scan(tiles, part[1]);
    const bool writer = blockIdx.x == 0;
#pragma unroll
    for (int i = 0; i < kPer; ++i) {
        const int e = kPer * tid + i;
        off[e] = row0;
        if (writer && e < a.experts) {
            a.offsets[e] = row0;
            if (e + 1 == a.experts) a.offsets[e + 1] = row0 + cnt[i];
            for (int r = 0; r < cnt[i]; r += a.tile_rows, ++tile0)
                if (tile0 < a.max_tiles) { a.tiles[2 * tile0] = e; a.tiles[2 * tile0 + 1] = r; }
        }
        row0 += cnt[i];
    }
    if (writer) {
        int total = 0;
        for (int i = 0; i < 4; ++i) total += part[1][i];
        // part[1] holds every wavefront's number of tiles
        for (int t = total + tid; t < a.max_tiles; t += kThreads) a.tiles[2 * t] = -1;
    }
    __syncthreads();
    const int64_t i = (int64_t)blockIdx.x * kThreads + tid;
    if (i >= a.choices) return;
    const int id = a.ids[i];
    if (id >= a.experts) {
        a.places[i] = -1;
        return;
    }
    const int place = off[id] + a.ranks[i];
    a.places[i] = place;
    a.row_token[place] = (int32_t)(i / a.top);
    a.row_expert[place] = id;
}

template <class T>
struct GemmArgs {
    const T* x; int64_t x_stride;
    const int32_t* row_token;              // row of x of every place, or nullptr: the place itself
    const int32_t* row_expert;
    const int32_t* offsets; const int32_t* tiles;
    const T* w; int64_t w_expert; int64_t w_stride;    // [expert][rows][k]
    int k, cols, up_row;                   // up_row > 0: columns of the result come from rows c (gate) and up_row + c (up)
    T* out; int64_t out_stride; int out_cols;          // columns from `cols` to out_cols are zero
    int32_t* zero; int num_zero;           // cleared by the launch
    int experts, max_tiles, col_blocks;
};

template <class T>
__device__ __forceinline__ void clear_counts(const GemmArgs<T>& a) {
    if (a.zero && blockIdx.x == 0)
        for (int i = threadIdx.x; i < a.num_zero; i += kThreads) a.zero[i] = 0;
}

// A workgroup: 128 rows of one expert x 128 rows of W (GATED: 64 gate rows and the same 64 up rows), k in steps of 64 through two LDS
// buffers.  Wavefront (wm, wn) has 64 rows x 64 rows of W as 4 x 4 tiles; with GATED, its first two tiles are gate and the other
// two up columns of the same place, so that the activation stays in registers.
constexpr int kBigRows = 128;
template <bool GATED>
__global__ void __launch_bounds__(kThreads, 2) moe_tile_kernel(GemmArgs<__bf16> a) {
    constexpr int kRow = 128 + 16, kMat = 128 * kRow;
    __shared__ __attribute__((aligned(16))) unsigned char lds[2][2 * kMat];
    clear_counts(a);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, n = lane & 15;
    // Workgroups go to the eight dies round-robin: each die gets a contiguous run of (tile, columns), columns fastest within
    // groups of tiles, so that the rows and weights it reads stay in its cache.
    const unsigned total = gridDim.x, id = blockIdx.x, die = id & 7u, per_die = total >> 3, extra = total & 7u;
    const unsigned unit = die * per_die + (die < extra ? die : extra) + (id >> 3);
    const int tile = (int)(unit / a.col_blocks), cb = (int)(unit % a.col_blocks);
    const int expert = a.tiles[2 * tile];
    if (expert < 0 || expert >= a.experts) return;
    const int first = a.offsets[expert] + a.tiles[2 * tile + 1], end = a.offsets[expert + 1];
    const int rows = end - first < kBigRows ? end - first : kBigRows;
    const __bf16* w = a.w + (int64_t)expert * a.w_expert;
    const int c0 = cb * (GATED ? 64 : 128);
    // unit i of this thread: row tid / 8 + 32 i of each tile, 16 bytes at column 8 (tid % 8)
    const int kc = 8 * (tid & 7);
    const __bf16* xs[4];
    const __bf16* ws[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int r = (tid >> 3) + 32 * i, xr = first + (r < rows ? r : rows - 1);
        xs[i] = a.x + (int64_t)(a.row_token ? a.row_token[xr] : xr) * a.x_stride;
        int col = GATED ? c0 + 32 * (r >> 6) + (r & 31) : c0 + r;
        col = col < a.cols ? col : a.cols - 1;
        ws[i] = w + (int64_t)(GATED && (r & 32) ? a.up_row + col : col) * a.w_stride;
    }
    u32x4_t xreg[4], wreg[4];
    auto fetch = [&](int k) {
        const bool in = k + kc < a.k;
        const int at = in ? k + kc : 0;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            xreg[i] = *reinterpret_cast<const u32x4_t*>(xs[i] + at);
            wreg[i] = *reinterpret_cast<const u32x4_t*>(ws[i] + at);
        }
    };
    auto put = [&](unsigned char* buf, int k) {
        const bool in = k + kc < a.k;                            // k is a multiple of eight
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int r = (tid >> 3) + 32 * i;
            *reinterpret_cast<u32x4_t*>(buf + r * kRow + 2 * kc) = in ? xreg[i] : u32x4_t{0u, 0u, 0u, 0u};
            *reinterpret_cast<u32x4_t*>(buf + kMat + r * kRow + 2 * kc) = in ? wreg[i] : u32x4_t{0u, 0u, 0u, 0u};
        }
    };
    const int wm = wave & 1, wn = wave >> 1;
    f32x4_t acc[4][4];                                           // [tile of W][tile of rows]
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    fetch(0);
    put(lds[0], 0);
    const int steps = (a.k + 63) / 64;
    if (steps > 1) fetch(64);
    for (int s = 0; s < steps; ++s) {
        __syncthreads();
        const unsigned char* buf = lds[s & 1];
        if (s + 1 < steps) put(lds[(s + 1) & 1], 64 * (s + 1));
        if (s + 2 < steps) fetch(64 * (s + 2));
#pragma unroll
        for (int k = 0; k < 2; ++k) {
            bf16x8_t xf[4], wf[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                xf[i] = *reinterpret_cast<const bf16x8_t*>(buf + (64 * wm + 16 * i + n) * kRow + 64 * k + 16 * g);
                wf[i] = *reinterpret_cast<const bf16x8_t*>(buf + kMat + (64 * wn + 16 * i + n) * kRow + 64 * k + 16 * g);
            }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[i], xf[j], acc[i][j], 0, 0, 0);
        }
    }
    // lane (g, n): row n of a row tile, columns 4 g + e
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int r = 64 * wm + 16 * j + n;
        if (r >= rows) continue;
        __bf16* o = a.out + (int64_t)(first + r) * a.out_stride;
#pragma unroll
        for (int i = 0; i < (GATED ? 2 : 4); ++i) {
            const int c = c0 + (GATED ? 32 : 64) * wn + 16 * i + 4 * g;
            bf16x4_t v;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                float x = acc[i][j][e];
                if constexpr (GATED) x = silu_f(x) * acc[i + 2][j][e];
                v[e] = (__bf16)(c + e < a.cols ? x : 0.f);
            }
            if (c + 4 <= a.out_cols) {
                *reinterpret_cast<bf16x4_t*>(o + c) = v;
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (c + e < a.out_cols) o[c + e] = v[e];
            }
        }
    }
}

// A workgroup of eight wavefronts: 256 rows of one expert x 256 rows of W (GATED: 128 gate rows and the same 128 up rows), k in steps
// of 64 (a multiple of which k is) through two LDS buffers that are filled from memory without passing through registers: the
// requests of the next step travel while this one is consumed.  Wavefront (wm, wn) has 128 rows x 64 rows of W as 8 x 4 tiles.
// A row of a buffer is eight units of 16 bytes, unit c at place c ^ (row % 8), so that reads of a column meet all banks.
constexpr int kBlockRows = 256, kBlockThreads = 512;
// (tiles, column blocks) that one die works on at a time: as many as it has compute units, and as square as column blocks of 256 allow
constexpr int kPatchTiles = 4, kPatchCols = 8, kPatch = kPatchTiles * kPatchCols;
template <bool GATED>
__global__ void __launch_bounds__(kBlockThreads, 2) moe_block_kernel(GemmArgs<__bf16> a) {
    constexpr int kMat = kBlockRows * 128, kBuf = 2 * kMat;      // bytes
    __shared__ __attribute__((aligned(1024))) unsigned char lds[2 * kBuf];
    if (a.zero && blockIdx.x == 0)
        for (int i = threadIdx.x; i < a.num_zero; i += kBlockThreads) a.zero[i] = 0;
    const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, n = lane & 15;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    // workgroups go to the eight dies round-robin, and so do the patches
    const unsigned seq = blockIdx.x >> 3, patch = seq / kPatch * 8u + (blockIdx.x & 7u), in_patch = seq % kPatch;
    const unsigned across = (unsigned)(a.col_blocks + kPatchCols - 1) / kPatchCols;
    const int tile = (int)(patch / across * kPatchTiles + in_patch % kPatchTiles);
    const int cb = (int)(patch % across * kPatchCols + in_patch / kPatchTiles);
    if (tile >= a.max_tiles || cb >= a.col_blocks) return;
    const int expert = a.tiles[2 * tile];
    if (expert < 0 || expert >= a.experts) return;
    const int first = a.offsets[expert] + a.tiles[2 * tile + 1], end = a.offsets[expert + 1];
    const int rows = end - first < kBlockRows ? end - first : kBlockRows;
    const int c0 = cb * (GATED ? 128 : 256);
    // load i of a wavefront fills rows 8 (4 wave + i) .. + 7: lane l place l % 8 of row l / 8
    uint32_t x_off[4], w_off[4], to[4];                          // bytes (checked on the host to fit)
    const uint32_t base = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) void*)lds;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int r = 8 * (4 * wave + i) + (lane >> 3), unit = (lane & 7) ^ (lane >> 3);
        const int xr = first + (r < rows ? r : rows - 1);
        x_off[i] = 2u * ((uint32_t)(a.row_token ? a.row_token[xr] : xr) * (uint32_t)a.x_stride + 8u * unit);
        int col = GATED ? c0 + 32 * (r >> 6) + (r & 31) : c0 + r;
        col = col < a.cols ? col : a.cols - 1;
        w_off[i] = 2u * ((uint32_t)(GATED && (r & 32) ? a.up_row + col : col) * (uint32_t)a.w_stride + 8u * unit);
        to[i] = __builtin_amdgcn_readfirstlane(base + (uint32_t)(1024 * (4 * wave + i)));
    }
    const __bf16* xs = a.x;
    const __bf16* ws = a.w + (int64_t)expert * a.w_expert;
    // Inline assembly, since the compiler would put a wait for all requests in front of every read of LDS.  Nothing else here uses M0.
    auto request = [&](uint32_t off, const __bf16* from, uint32_t at) {
        __asm__ volatile("s_mov_b32 m0, %2\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %0, %1" :: "v"(off), "s"(from), "s"(at) : "memory", "m0");
    };
    auto fetch = [&](int s, uint32_t buf) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            request(x_off[i], xs + 64 * s, to[i] + buf);
            request(w_off[i], ws + 64 * s, to[i] + buf + kMat);
        }
    };
    const int wm = wave & 1, wn = wave >> 1;
    const bool live = 128 * wm < rows;
    f32x4_t acc[4][8];                                           // [tile of W][tile of rows]
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 8; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const int steps = a.k / 64;
    fetch(0, 0);
    const int unit0 = n * 128 + 16 * (g ^ (n & 7));
    for (int s = 0; s < steps; ++s) {
        // this wavefront's requests have landed; behind the barrier everybody's have, and nobody reads the other buffer any more
        __builtin_amdgcn_s_waitcnt(0x0F70);
        __syncthreads();
        if (s + 1 < steps) fetch(s + 1, (uint32_t)((s + 1) & 1) * kBuf);
        if (!live) continue;
        const unsigned char* xb = lds + (s & 1) * kBuf + 128 * 128 * wm;
        const unsigned char* wb = lds + (s & 1) * kBuf + kMat + 64 * 128 * wn;
#pragma unroll
        for (int k = 0; k < 2; ++k) {
            const int at = unit0 ^ (64 * k);
            bf16x8_t xf[8], wf[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) wf[i] = *reinterpret_cast<const bf16x8_t*>(wb + at + 2048 * i);
#pragma unroll
            for (int j = 0; j < 8; ++j) xf[j] = *reinterpret_cast<const bf16x8_t*>(xb + at + 2048 * j);
#pragma unroll
            for (int j = 0; j < 8; ++j)
#pragma unroll
                for (int i = 0; i < 4; ++i) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[i], xf[j], acc[i][j], 0, 0, 0);
        }
    }
    // lane (g, n): row n of a row tile, columns 4 g + e
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        const int r = 128 * wm + 16 * j + n;
        if (r >= rows) continue;
        __bf16* o = a.out + (int64_t)(first + r) * a.out_stride;
#pragma unroll
        for (int i = 0; i < (GATED ? 2 : 4); ++i) {
            const int c = c0 + (GATED ? 32 : 64) * wn + 16 * i + 4 * g;
            bf16x4_t v;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                float x = acc[i][j][e];
                if constexpr (GATED) x = silu_f(x) * acc[i + 2][j][e];
                v[e] = (__bf16)(c + e < a.cols ? x : 0.f);
            }
            if (c + 4 <= a.out_cols) *reinterpret_cast<bf16x4_t*>(o + c) = v;       // out_cols is a multiple of eight
        }
    }
}

// A workgroup: 16 rows of one expert x 32 rows of W (GATED: 16 gate and 16 up); wavefront w takes the k-steps w, w + 4, ...
constexpr int kSmallRows = 16;
template <bool GATED>
__global__ void __launch_bounds__(kThreads) moe_row_kernel(GemmArgs<__bf16> a) {
    __shared__ float part[4][2][16][17];
    clear_counts(a);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, n = lane & 15;
    const int tile = blockIdx.x / a.col_blocks, cb = blockIdx.x % a.col_blocks;
    const int expert = a.tiles[2 * tile];
    if (expert < 0 || expert >= a.experts) return;
    const int first = a.offsets[expert] + a.tiles[2 * tile + 1], end = a.offsets[expert + 1];
    const int rows = end - first < kSmallRows ? end - first : kSmallRows;
    const int c0 = cb * (GATED ? 16 : 32), xr = first + (n < rows ? n : rows - 1);
    const __bf16* x = a.x + (int64_t)(a.row_token ? a.row_token[xr] : xr) * a.x_stride;
    const __bf16* w = a.w + (int64_t)expert * a.w_expert;
    const __bf16* wr[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        int col = c0 + n + (GATED ? 0 : 16 * i);
        col = col < a.cols ? col : a.cols - 1;
        wr[i] = w + (int64_t)(GATED && i ? a.up_row + col : col) * a.w_stride;
    }
    f32x4_t acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    constexpr int kAhead = 4;
    for (int k0 = 32 * wave; k0 < a.k; k0 += 128 * kAhead) {
        bf16x8_t xf[kAhead], wf[kAhead][2];
#pragma unroll
        for (int j = 0; j < kAhead; ++j) {
            const int k = k0 + 128 * j + 8 * g;
            const int at = k < a.k ? k : 0;
            xf[j] = *reinterpret_cast<const bf16x8_t*>(x + at);
#pragma unroll
            for (int i = 0; i < 2; ++i) wf[j][i] = *reinterpret_cast<const bf16x8_t*>(wr[i] + at);
        }
#pragma unroll
        for (int j = 0; j < kAhead; ++j) {
            if (k0 + 128 * j + 8 * g >= a.k) xf[j] = bf16x8_t{};
#pragma unroll
            for (int i = 0; i < 2; ++i) acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[j][i], xf[j], acc[i], 0, 0, 0);
        }
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) part[wave][i][n][4 * g + e] = acc[i][e];
    __syncthreads();
    const int r = tid >> 4, c = tid & 15;
    if (r >= rows) return;
    float v[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) v[i] = part[0][i][r][c] + part[1][i][r][c] + part[2][i][r][c] + part[3][i][r][c];
    __bf16* o = a.out + (int64_t)(first + r) * a.out_stride + c0 + c;
    if constexpr (GATED) {
        if (c0 + c < a.out_cols) o[0] = (__bf16)(c0 + c < a.cols ? silu_f(v[0]) * v[1] : 0.f);
    } else {
#pragma unroll
        for (int i = 0; i < 2; ++i)
            if (c0 + 16 * i + c < a.out_cols) o[16 * i] = (__bf16)(c0 + 16 * i + c < a.cols ? v[i] : 0.f);
    }
}

// one wavefront per (place, four columns)
template <class T, bool GATED>
__global__ void __launch_bounds__(kThreads) moe_any_kernel(GemmArgs<T> a) {
    clear_counts(a);
    const int lane = threadIdx.x & 63;
    const int64_t place = blockIdx.x / a.col_blocks;
    if (place >= a.offsets[a.experts]) return;
    const int expert = a.row_expert[place];
    const T* x = a.x + (int64_t)(a.row_token ? a.row_token[place] : place) * a.x_stride;
    const T* w = a.w + (int64_t)expert * a.w_expert;
    for (int i = 0; i < 4; ++i) {
        const int c = (blockIdx.x % a.col_blocks) * 16 + (threadIdx.x >> 6) * 4 + i;
        if (c >= a.out_cols) break;
        float s = 0.f, u = 0.f;
        if (c < a.cols)
            for (int k = lane; k < a.k; k += 64) {
                s += (float)x[k] * (float)w[(int64_t)c * a.w_stride + k];
                if (GATED) u += (float)x[k] * (float)w[(int64_t)(a.up_row + c) * a.w_stride + k];
            }
        s = wave_sum(s);
        if (GATED) s = silu_f(s) * wave_sum(u);
        if (lane == 0) a.out[place * a.out_stride + c] = (T)s;
    }
}

bool size_in(int64_t v, int64_t lo, int64_t hi) { return v >= lo && v <= hi; }

template <class T>
int gemm(GemmArgs<T>& a, bool gated, int tile_rows, int64_t max_places, hipStream_t st) {
    const dim3 block(kThreads);
    int64_t grid;
    if constexpr (sizeof(T) == 2) {
        if (tile_rows == kBlockRows) {
            a.col_blocks = (a.out_cols + (gated ? 127 : 255)) / (gated ? 128 : 256);
            const int64_t patches = (int64_t)((a.max_tiles + kPatchTiles - 1) / kPatchTiles) * ((a.col_blocks + kPatchCols - 1) / kPatchCols);
            grid = (patches + 7) / 8 * 8 * kPatch;
            if (grid > 0x7fffffff) return INFER_KV_EINVAL;
            if (gated) hipLaunchKernelGGL((moe_block_kernel<true>), dim3((unsigned)grid), dim3(kBlockThreads), 0, st, a);
            else hipLaunchKernelGGL((moe_block_kernel<false>), dim3((unsigned)grid), dim3(kBlockThreads), 0, st, a);
            return (int)hipGetLastError();
        }
        if (tile_rows == kBigRows || tile_rows == kSmallRows) {
            const int per = tile_rows == kBigRows ? (gated ? 64 : 128) : (gated ? 16 : 32);
            a.col_blocks = (a.out_cols + per - 1) / per;
            grid = (int64_t)a.max_tiles * a.col_blocks;
            if (grid > 0x7fffffff) return INFER_KV_EINVAL;
            if (tile_rows == kBigRows) {
                if (gated) hipLaunchKernelGGL((moe_tile_kernel<true>), dim3((unsigned)grid), block, 0, st, a);
                else hipLaunchKernelGGL((moe_tile_kernel<false>), dim3((unsigned)grid), block, 0, st, a);
            } else {
                if (gated) hipLaunchKernelGGL((moe_row_kernel<true>), dim3((unsigned)grid), block, 0, st, a);
                else hipLaunchKernelGGL((moe_row_kernel<false>), dim3((unsigned)grid), block, 0, st, a);
            }
            return (int)hipGetLastError();
        }
    }
    a.col_blocks = (a.out_cols + 15) / 16;
    grid = max_places * a.col_blocks;
    if (grid > 0x7fffffff) return INFER_KV_EINVAL;
    if (gated) hipLaunchKernelGGL((moe_any_kernel<T, true>), dim3((unsigned)grid), block, 0, st, a);
    else hipLaunchKernelGGL((moe_any_kernel<T, false>), dim3((unsigned)grid), block, 0, st, a);
    return (int)hipGetLastError();
}

// rows per tile: 0 where only the any-size kernels serve
int rows_per_tile(int elem, int64_t n, int64_t width, int64_t ff_pad, int64_t experts, int64_t top) {
    if (elem != INFER_ELEM_BF16 || width % 8 || ff_pad % 8) return 0;
    if (n * top <= 24 * experts) return kSmallRows;
    // large blocks pay when most of them are full; their offsets are 32 bits
    const int64_t far = 1ll << 31;
    const bool fits = width % 64 == 0 && ff_pad % 64 == 0 && n * width < far && n * top * ff_pad < far && 2 * ff_pad * width < far;
    return fits && n * top >= 512 * experts ? kBlockRows : kBigRows;
}

}  // namespace

// places (rows of the two products) and tiles of a step of n tokens, and the rows per tile: out[3]
extern "C" int infer_moe_layout(int elem, int64_t n, int64_t width, int64_t ff_pad, int64_t experts, int64_t top, int64_t* out) {
    if (n < 0 || width < 1 || experts < 1 || top < 1 || !out) return INFER_KV_EINVAL;
    const int per = rows_per_tile(elem, n, width, ff_pad, experts, top);
    out[0] = n * top;
    out[1] = per ? n * top / per + (experts < n * top ? experts : n * top) : 1;
    out[2] = per;
    return INFER_KV_OK;
}

extern "C" int infer_moe(int elem, const void* h, int64_t h_stride, const void* router, const float* correction, int64_t n, int64_t width,
                         int64_t experts, int64_t identity, int64_t top, int64_t groups, int64_t keep, float scale, const void* gate_up,
                         const void* down, int64_t ff, int64_t ff_pad, int32_t* counts, int32_t* ids, float* weights, int32_t* ranks,
                         int32_t* places, int32_t* row_token, int32_t* row_expert, int32_t* offsets, int32_t* tiles, int64_t max_tiles,
                         void* act, void* out, int64_t max_places, void* stream) {
    const int64_t all = experts + identity;
    if (!size_in(n, 0, 1 << 26) || !size_in(width, 1, 1 << 20) || !size_in(experts, 1, kMaxExperts) || identity < 0 || all > kMaxExperts ||
        !size_in(top, 1, 64) || top > all || !size_in(groups, 1, all) || all % groups || !size_in(keep, 1, groups) ||
        keep * (all / groups) < top || !size_in(ff, 1, 1 << 20) || ff_pad < ff || h_stride < width)
        return INFER_KV_EINVAL;
    if (n == 0) return INFER_KV_OK;
    int64_t layout[3];
    infer_moe_layout(elem, n, width, ff_pad, experts, top, layout);
    if (!h || !router || !gate_up || !down || !counts || !ids || !weights || !ranks || !places || !row_token || !row_expert || !offsets ||
        !tiles || !act || !out || max_places < layout[0] || max_tiles < layout[1] || n * top > 0x7fffffff)
        return INFER_KV_EINVAL;
    hipStream_t st = (hipStream_t)stream;
    auto go = [&](auto zero) -> int {
        using T = decltype(zero);
        const RouteArgs<T> r{(const T*)h, h_stride, (const T*)router, correction, (int)width, (int)all, (int)experts, (int)top, (int)groups,
                             (int)keep, scale, ids, weights, ranks, counts, (int)n};
        const bool aligned = width % 8 == 0 && h_stride % 8 == 0 && ptr_aligned(h, 16) && ptr_aligned(gate_up, 16) && ptr_aligned(down, 16) &&
                             ptr_aligned(act, 16) && ptr_aligned(out, 16);
        bool routed = false;
        if constexpr (sizeof(T) == 2) {
            if (aligned && width % 32 == 0 && all <= 256 && ptr_aligned(router, 16)) {
                if (all <= 16) launch_route<1>(r, st);
                else if (all <= 64) launch_route<4>(r, st);
                else if (all <= 128) launch_route<8>(r, st);
                else launch_route<16>(r, st);
                routed = true;
            }
        }
        if (!routed) hipLaunchKernelGGL((moe_route_any_kernel<T>), dim3((unsigned)((n + 3) / 4)), dim3(kThreads), 0, st, r);
        const int tile_rows = aligned ? (int)layout[2] : 0;
        if (tile_rows == kBlockRows && n * h_stride >= (1ll << 31)) return INFER_KV_EUNSUPPORTED;
        const int64_t choices = n * top;
        const ScatterArgs s{ids, ranks, counts, (int)experts, (int)top, tile_rows ? tile_rows : kBigRows, (int)max_tiles, choices, places, row_token,
                            row_expert, offsets, tiles};
        hipLaunchKernelGGL(moe_scatter_kernel, dim3((unsigned)((choices + kThreads - 1) / kThreads)), dim3(kThreads), 0, st, s);
        GemmArgs<T> up{(const T*)h, h_stride, row_token, row_expert, offsets, tiles, (const T*)gate_up, 2 * ff * width, width, (int)width, (int)ff,
                       (int)ff, (T*)act, ff_pad, (int)ff_pad, counts, (int)experts, (int)experts, (int)max_tiles, 0};
        int rc = gemm(up, true, tile_rows, max_places, st);
        if (rc) return rc;
        GemmArgs<T> dn{(const T*)act, ff_pad, nullptr, row_expert, offsets, tiles, (const T*)down, width * ff_pad, ff_pad, (int)ff_pad, (int)width,
                       0, (T*)out, width, (int)width, nullptr, 0, (int)experts, (int)max_tiles, 0};
        return gemm(dn, false, tile_rows, max_places, st);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}
