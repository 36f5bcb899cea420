// Attention whose heads mix their softmax weights, query row by query row over pages of tiles (tile_pages.h), for gfx950 (MI355X).
//
//     w_h(j) = e^{s_h(j)} / (1 + sum_j' e^{s_h(j')}) ,   o_h = c sum_j (sum_g T[h][g] w_g(j)) v_j
//
// with s = scale q.k over the keys that the row sees, v of the key/value head that head h shares with its group, and T a matrix over all
// heads.  The one in the denominator is a sink: a score of zero that belongs to no key.  (A row is a token: decoded tokens and the
// tokens of short prompt portions; long portions run in talking_prefill.hip.)
//
// The mixture needs complete denominators of all heads, so keys and values are read by two kernels, with the scores (float32, in units
// of log2) in memory in between:
//   talk_scores_kernel   scores, and per (row, split of the keys, head) their maximum and the sum of their powers
//   talk_values_kernel   weights from the scores of all heads, mixed, times the values; splits of the keys are added up by
//   talk_merge_kernel
//   talk_scores_any_kernel, talk_values_any_kernel   the same for any size and element type
#include "elem.h"
#include "pieces.h"
#include "tile_pages.h"

namespace {

constexpr int kTile = kTileTokens;
constexpr int kWaves = 4;
constexpr float kLow = -1e30f;            // a maximum before any key was seen; finite, since hidden scores are -inf

template <class T>
struct TalkArgs {
    const T* qx;                          // [rows][heads][key_pad]
    const T* keys; const T* values;       // [blocks][kv_heads][tiles of block_size tokens], key_pad and vdim_pad entries per token
    int key_pad, vdim_pad;
    const int32_t* bt; int64_t bt_stride; int table_cols, block_size, num_blocks;
    const int32_t* row_seq;               // block-table row of each query row; nullptr: the query row itself
    const int32_t* ctx;                   // keys each query row sees
    int rows, heads, kv_heads, splits;
    float scale_log2;
    const T* talk;                        // [heads][heads]
    float out_scale;
    T* out; int64_t out_row; int vdim;    // [rows][heads * vdim]
    float* scores; int64_t key_cap;       // [rows][heads][key_cap]
    float* ml;                            // [rows][splits][heads][max, sum]
    float* part;                          // [rows][splits][heads][vdim_pad], if splits > 1
    unsigned groups;                      // head groups of the launch
};

template <class T>
__device__ __forceinline__ int visible_keys(const TalkArgs<T>& a, int row) {
    const int len = a.ctx[row], cap = a.table_cols * a.block_size;
    const int n = len < cap ? len : cap;  // a corrupt length runs neither past the table row nor past the scores
    return n < a.key_cap ? n : (int)a.key_cap;
}
template <class T>
__device__ __forceinline__ const int32_t* table_of(const TalkArgs<T>& a, int row) {
    return a.bt + (int64_t)(a.row_seq ? a.row_seq[row] : row) * a.bt_stride;
}
template <class T>
__device__ __forceinline__ int block_id(const TalkArgs<T>& a, const int32_t* bt, int col) {
    const int b = bt[col < a.table_cols ? col : a.table_cols - 1];
    return b < 0 ? 0 : (b >= a.num_blocks ? a.num_blocks - 1 : b);
}
// tiles of a row and how many of them a split has
template <class T>
__device__ __forceinline__ int tiles_per_split(const TalkArgs<T>& a, int tiles) { return (tiles + a.splits - 1) / a.splits; }
template <class T>
__device__ __forceinline__ int used_splits(const TalkArgs<T>& a, int len) {
    const int tiles = (len + kTile - 1) / kTile, per = tiles_per_split(a, tiles);
    return per > 0 ? (tiles + per - 1) / per : 0;
}
// log2 of a head's denominator, the sink among its terms
template <class T>
__device__ __forceinline__ float log_denominator(const TalkArgs<T>& a, int row, int h, int used) {
    const float* ml = a.ml + ((int64_t)row * a.splits * a.heads + h) * 2;
    const int64_t next = 2 * (int64_t)a.heads;
    float m = 0.f;
    for (int s = 0; s < used; ++s) m = fmaxf(m, ml[s * next]);
    float sum = exp2f(-m);
    for (int s = 0; s < used; ++s) sum += ml[s * next + 1] * exp2f(ml[s * next] - m);
    return m + log2f(sum);
}
// where the tile of a key begins, in tokens of all blocks of one head; the key's place in it
template <class T>
__device__ __forceinline__ int64_t tile_of(const TalkArgs<T>& a, const int32_t* bt, int kvh, int key, int& token) {
    const int col = key / a.block_size, off = key - col * a.block_size;
    token = off % kTile;
    return ((int64_t)block_id(a, bt, col) * a.kv_heads + kvh) * a.block_size + off - token;
}
__device__ __forceinline__ void join_max_sum(float& m, float& l, float m2, float l2) {
    const float top = fmaxf(m, m2);
    l = l * exp2f(m - top) + l2 * exp2f(m2 - top);
    m = top;
}

// ------------------------------------------------------------------ any size
// One workgroup per (query row, head); wavefront w takes keys w, w + 4, ...
template <class T, int NC>
__global__ void __launch_bounds__(256) talk_scores_any_kernel(TalkArgs<T> a) {
    __shared__ float sm[kWaves], sl[kWaves];
    const int row = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int len = visible_keys(a, row), kvh = h / (a.heads / a.kv_heads);
    const int32_t* bt = table_of(a, row);
    const T* qr = a.qx + ((int64_t)row * a.heads + h) * a.key_pad;
    float* out = a.scores + ((int64_t)row * a.heads + h) * a.key_cap;
    float q[NC];
#pragma unroll
    for (int i = 0; i < NC; ++i) q[i] = lane + 64 * i < a.key_pad ? (float)qr[lane + 64 * i] * a.scale_log2 : 0.f;
    float m = kLow, l = 0.f;
    for (int key = wave; key < len; key += kWaves) {
        int token;
        const T* kr = a.keys + tile_of(a, bt, kvh, key, token) * a.key_pad;
        float s = 0.f;
#pragma unroll
        for (int i = 0; i < NC; ++i)
            if (lane + 64 * i < a.key_pad) s += q[i] * (float)kr[tile_key_entry(token, lane + 64 * i)];
        s = wave_sum(s);
        if (lane == 0) out[key] = s;
        join_max_sum(m, l, s, 1.f);
    }
    if (lane == 0) { sm[wave] = m; sl[wave] = l; }
    __syncthreads();
    if (threadIdx.x == 0) {
        for (int i = 1; i < kWaves; ++i) join_max_sum(m, l, sm[i], sl[i]);
        a.ml[2 * ((int64_t)row * a.heads + h)] = m;
        a.ml[2 * ((int64_t)row * a.heads + h) + 1] = l;
    }
}

// One workgroup per (query row, head): mixed weights of 256 keys at a time, one by every thread, then the values.  COLS: columns per
// thread; the threads are `lanes` columns by 256 / lanes parts of the keys.
template <class T, int COLS>
__global__ void __launch_bounds__(256) talk_values_any_kernel(TalkArgs<T> a, int lanes) {
    extern __shared__ float sh[];
    float* lse = sh;                                 // [heads]
    float* mix = lse + a.heads;                      // [heads]
    float* p = mix + a.heads;                        // [256]
    float* red = p + 256;                            // [256]
    const int row = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    const int len = visible_keys(a, row), kvh = h / (a.heads / a.kv_heads);
    const int32_t* bt = table_of(a, row);
    for (int g = tid; g < a.heads; g += 256) {
        lse[g] = log_denominator(a, row, g, used_splits(a, len));
        mix[g] = (float)a.talk[(int64_t)h * a.heads + g];
    }
    const int c = tid % lanes, part = tid / lanes, parts = 256 / lanes;
    float o[COLS];
#pragma unroll
    for (int i = 0; i < COLS; ++i) o[i] = 0.f;
    for (int k0 = 0; k0 < len; k0 += 256) {
        __syncthreads();
        const int mine = k0 + tid;
        if (mine < len) {
            const float* s = a.scores + (int64_t)row * a.heads * a.key_cap + mine;
            float w = 0.f;
            for (int g = 0; g < a.heads; ++g) w += mix[g] * exp2f(s[g * a.key_cap] - lse[g]);
            p[tid] = w;
        }
        __syncthreads();
        const int count = len - k0 < 256 ? len - k0 : 256;
        for (int k = part; k < count; k += parts) {
            int token;
            const T* vr = a.values + tile_of(a, bt, kvh, k0 + k, token) * a.vdim_pad;
#pragma unroll
            for (int i = 0; i < COLS; ++i)
                if (c + lanes * i < a.vdim) o[i] += p[k] * (float)vr[tile_value_entry(token, c + lanes * i)];
        }
    }
#pragma unroll
    for (int i = 0; i < COLS; ++i) {
        __syncthreads();
        red[tid] = o[i];
        __syncthreads();
        if (part == 0 && c + lanes * i < a.vdim) {
            float x = 0.f;
            for (int k = 0; k < parts; ++k) x += red[k * lanes + c];
            a.out[(int64_t)row * a.out_row + (int64_t)h * a.vdim + c + lanes * i] = (T)(x * a.out_scale);
        }
    }
}

// ------------------------------------------------------------------ MFMA forms
// What a workgroup works on: 16 MT heads of one key/value head, one query row, a run of 32-key tiles (a split).  Workgroups go to the
// eight dies round-robin: the head groups of one (row, split) are given to one die, whose second-level cache then serves the scores
// that all of them read.
template <int MT>
struct Unit {
    int row, split, kvh, head0, head_end, len, t0, t1;
    bool exists;
    __device__ __forceinline__ Unit(const TalkArgs<__bf16>& a) {
        const unsigned die = blockIdx.x & 7u, turn = blockIdx.x >> 3, unit = turn / a.groups * 8u + die;
        exists = unit < (unsigned)(a.rows * a.splits);
        if (!exists) return;
        split = (int)(unit % (unsigned)a.splits);
        row = (int)(unit / (unsigned)a.splits);
        const int shared = a.heads / a.kv_heads, per_kv = (shared + 16 * MT - 1) / (16 * MT), group = (int)(turn % a.groups);
        kvh = group / per_kv;
        head0 = kvh * shared + (group - kvh * per_kv) * 16 * MT;
        head_end = (kvh + 1) * shared;
        len = visible_keys(a, row);
        const int tiles = (len + kTile - 1) / kTile, per = tiles_per_split(a, tiles);
        t0 = split * per;
        t1 = t0 + per < tiles ? t0 + per : tiles;
    }
};

// The tiles t, t + 4, ... of one wavefront: a tile lies in one block, whose id is looked up one step ahead.
struct TileWalk {
    int tiles_per_block, col, in_block, next_id;
    __device__ __forceinline__ TileWalk(const TalkArgs<__bf16>& a, const int32_t* bt, int t) {
        tiles_per_block = a.block_size / kTile;
        col = t / tiles_per_block;
        in_block = t - col * tiles_per_block;
        next_id = block_id(a, bt, col);
    }
    // the tile's number among the tiles of all blocks of one head; then moves on
    __device__ __forceinline__ int64_t next(const TalkArgs<__bf16>& a, const int32_t* bt, int kvh) {
        const int64_t at = ((int64_t)next_id * a.kv_heads + kvh) * tiles_per_block + in_block;
        in_block += kWaves;
        while (in_block >= tiles_per_block) { in_block -= tiles_per_block; ++col; }
        next_id = block_id(a, bt, col);
        return at;
    }
};

// S^T[key, head] = K[key, :] . Q^T; every wavefront has tiles of its own and reads their keys straight into operands.
template <int MT, int KS>
__global__ void __launch_bounds__(256) talk_scores_kernel(TalkArgs<__bf16> a) {
    __shared__ float sm[kWaves][16 * MT], sl[kWaves][16 * MT];
    const Unit<MT> u(a);
    if (!u.exists || u.t0 >= u.t1) return;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, n = lane & 15;
    const int32_t* bt = table_of(a, u.row);
    bf16x8_t q[MT][KS];
    float* to[MT];
#pragma unroll
    for (int i = 0; i < MT; ++i) {
        const int h = u.head0 + 16 * i + n;
        const int64_t at = (int64_t)u.row * a.heads + (h < u.head_end ? h : u.head0);
        to[i] = h < u.head_end ? a.scores + at * a.key_cap + 8 * g : nullptr;
#pragma unroll
        for (int j = 0; j < KS; ++j) {
            q[i][j] = bf16x8_t{};
            if (32 * j < a.key_pad) q[i][j] = *reinterpret_cast<const bf16x8_t*>(a.qx + at * a.key_pad + 32 * j + 8 * g);
        }
    }
    const int k_lane = tile_key_entry(tile_row_token(n, 0), 8 * g);
    int k_step[KS];                                   // k-steps behind the size repeat the first one, which meets zeros
#pragma unroll
    for (int j = 0; j < KS; ++j) k_step[j] = tile_key_entry(0, 32 * j < a.key_pad ? 32 * j : 0);
    float m[MT], l[MT];
#pragma unroll
    for (int i = 0; i < MT; ++i) { m[i] = kLow; l[i] = 0.f; }
    bf16x8_t kf[2][KS];
    TileWalk walk(a, bt, u.t0 + wave);
    auto fetch = [&]() {
        const __bf16* src = a.keys + walk.next(a, bt, u.kvh) * kTile * a.key_pad + k_lane;
#pragma unroll
        for (int x = 0; x < 2; ++x)
#pragma unroll
            for (int j = 0; j < KS; ++j) kf[x][j] = *reinterpret_cast<const bf16x8_t*>(src + k_step[j] + tile_key_entry(tile_row_token(0, x), 0));
    };
    if (u.t0 + wave < u.t1) fetch();
    for (int t = u.t0 + wave; t < u.t1; t += kWaves) {
        f32x4_t s[MT][2];
#pragma unroll
        for (int i = 0; i < MT; ++i)
#pragma unroll
            for (int x = 0; x < 2; ++x) {
                s[i][x] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int j = 0; j < KS; ++j) s[i][x] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[x][j], q[i][j], s[i][x], 0, 0, 0);
            }
        if (t + kWaves < u.t1) fetch();
        const int left = u.len - t * kTile - 8 * g;   // of this lane's keys 4 x + e those below `left` exist
#pragma unroll
        for (int i = 0; i < MT; ++i) {
            float top = m[i];
#pragma unroll
            for (int x = 0; x < 2; ++x) {
                s[i][x] *= a.scale_log2;
                if (to[i]) *reinterpret_cast<f32x4_t*>(to[i] + (int64_t)t * kTile + 4 * x) = s[i][x];
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    if (4 * x + e >= left) s[i][x][e] = -INFINITY;
                    top = fmaxf(top, s[i][x][e]);
                }
            }
            float sum = l[i] * __builtin_amdgcn_exp2f(m[i] - top);
#pragma unroll
            for (int x = 0; x < 2; ++x)
#pragma unroll
                for (int e = 0; e < 4; ++e) sum += __builtin_amdgcn_exp2f(s[i][x][e] - top);
            l[i] = sum;
            m[i] = top;
        }
    }
#pragma unroll
    for (int i = 0; i < MT; ++i) {
        join_max_sum(m[i], l[i], __shfl_xor(m[i], 16, 64), __shfl_xor(l[i], 16, 64));
        join_max_sum(m[i], l[i], __shfl_xor(m[i], 32, 64), __shfl_xor(l[i], 32, 64));
        if (g == 0) { sm[wave][16 * i + n] = m[i]; sl[wave][16 * i + n] = l[i]; }
    }
    __syncthreads();
    const int h = u.head0 + (int)threadIdx.x;
    if (threadIdx.x < 16 * MT && h < u.head_end) {
        float mt = sm[0][threadIdx.x], lt = sl[0][threadIdx.x];
#pragma unroll
        for (int w = 1; w < kWaves; ++w) join_max_sum(mt, lt, sm[w][threadIdx.x], sl[w][threadIdx.x]);
        float* ml = a.ml + (((int64_t)u.row * a.splits + u.split) * a.heads + h) * 2;
        ml[0] = mt;
        ml[1] = lt;
    }
}

// Every wavefront has tiles of its own and reads their values straight into operands:
//   P'^T[key, head] = W^T[key, g] . T^T[g, head]     weights of all heads g as two bf16 pieces each (2^-17), KH k-steps of 32 heads
//   O^T[v, head]   += V^T[v, key] . P'^T[key, head]
// A lane's eight results of the first product are the eight consecutive keys that the second one wants from it (tile_row_token).
template <int MT, int KH, int NT>
__global__ void __launch_bounds__(256) talk_values_kernel(TalkArgs<__bf16> a) {
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];
    __shared__ float lse[32 * KH];
    const Unit<MT> u(a);
    if (!u.exists || (u.t0 >= u.t1 && (a.splits > 1 || u.len > 0))) return;       // the merge knows which splits are empty
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), g = lane >> 4, n = lane & 15;
    const int32_t* bt = table_of(a, u.row);
    int v_tile[NT];                                   // value tiles behind the size repeat the first one and are not stored
#pragma unroll
    for (int v = 0; v < NT; ++v) v_tile[v] = tile_value_entry(0, 16 * v < a.vdim_pad ? 16 * v : 0);
    bf16x8_t vf[NT];
    float sreg[KH][2][8];
    const float* src_s[KH][8];
#pragma unroll
    for (int s = 0; s < KH; ++s)
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const int from = 32 * s + 8 * g + e;
            src_s[s][e] = a.scores + ((int64_t)u.row * a.heads + (from < a.heads ? from : a.heads - 1)) * a.key_cap + tile_row_token(n, 0);
        }
    TileWalk walk(a, bt, u.t0 + wave);
    auto fetch = [&](int t) {
        const __bf16* src = a.values + walk.next(a, bt, u.kvh) * kTile * a.vdim_pad + tile_value_entry(8 * g, n);
#pragma unroll
        for (int s = 0; s < KH; ++s)
#pragma unroll
            for (int x = 0; x < 2; ++x)
#pragma unroll
                for (int e = 0; e < 8; ++e) sreg[s][x][e] = src_s[s][e][(int64_t)t * kTile + 4 * x];
#pragma unroll
        for (int v = 0; v < NT; ++v) vf[v] = *reinterpret_cast<const bf16x8_t*>(src + v_tile[v]);
    };
    if (u.t0 + wave < u.t1) fetch(u.t0 + wave);
    const int used = used_splits(a, u.len);
    if (tid < 32 * KH) lse[tid] = tid < a.heads ? log_denominator(a, u.row, tid, used) : INFINITY;     // no such head: weight zero
    bf16x8_t tf[MT][KH];
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
        for (int s = 0; s < KH; ++s)
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const int h = u.head0 + 16 * i + n, from = 32 * s + 8 * g + e;
                tf[i][s][e] = h < u.head_end && from < a.heads ? a.talk[(int64_t)h * a.heads + from] : (__bf16)0.f;
            }
    __syncthreads();
    float den[KH][8];
#pragma unroll
    for (int s = 0; s < KH; ++s)
#pragma unroll
        for (int e = 0; e < 8; ++e) den[s][e] = lse[32 * s + 8 * g + e];
    f32x4_t acc[MT][NT];
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
        for (int v = 0; v < NT; ++v) acc[i][v] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int t = u.t0 + wave; t < u.t1; t += kWaves) {
        f32x4_t mixed[MT][2];
        const int left = u.len - t * kTile;
#pragma unroll
        for (int x = 0; x < 2; ++x) {
#pragma unroll
            for (int i = 0; i < MT; ++i) mixed[i][x] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int s = 0; s < KH; ++s) {
                float w[8];
#pragma unroll
                for (int e = 0; e < 8; ++e)
                    w[e] = tile_row_token(n, x) < left ? __builtin_amdgcn_exp2f(sreg[s][x][e] - den[s][e]) : 0.f;
                bf16x8_t wf[2];
                split_frags<2>(w, wf);
#pragma unroll
                for (int i = 0; i < MT; ++i)
#pragma unroll
                    for (int k = 1; k >= 0; --k) mixed[i][x] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[k], tf[i][s], mixed[i][x], 0, 0, 0);
            }
        }
        bf16x8_t pb[MT];
#pragma unroll
        for (int i = 0; i < MT; ++i)
#pragma unroll
            for (int e = 0; e < 8; ++e) pb[i][e] = (__bf16)mixed[i][e >> 2][e & 3];
        if (left < kTile)                             // values behind the last one may be anything
#pragma unroll
            for (int v = 0; v < NT; ++v)
#pragma unroll
                for (int e = 0; e < 8; ++e)
                    if (8 * g + e >= left) vf[v][e] = (__bf16)0.f;
#pragma unroll
        for (int v = 0; v < NT; ++v)
#pragma unroll
            for (int i = 0; i < MT; ++i) acc[i][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[v], pb[i], acc[i][v], 0, 0, 0);
        if (t + kWaves < u.t1) fetch(t + kWaves);
    }
    // ---- the wavefronts' sums, 16 heads at a time; columns behind the size are never stored
    f32x4_t* red = reinterpret_cast<f32x4_t*>(lds);   // [kWaves][NT][64]
#pragma unroll
    for (int i = 0; i < MT; ++i) {
        __syncthreads();
#pragma unroll
        for (int v = 0; v < NT; ++v) red[(wave * NT + v) * 64 + lane] = acc[i][v];
        __syncthreads();
        const int h = u.head0 + 16 * i + n;
#pragma unroll
        for (int v = 0; v < NT; ++v) {
            if (v % kWaves != wave || h >= u.head_end || 16 * v >= a.vdim_pad) continue;
            f32x4_t x = red[v * 64 + lane];
#pragma unroll
            for (int w = 1; w < kWaves; ++w) x += red[(w * NT + v) * 64 + lane];
            const int c = 16 * v + 4 * g;
            if (a.splits > 1) {
                *reinterpret_cast<f32x4_t*>(a.part + (((int64_t)u.row * a.splits + u.split) * a.heads + h) * a.vdim_pad + c) = x;
                continue;
            }
            __bf16* o = a.out + (int64_t)u.row * a.out_row + (int64_t)h * a.vdim;
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (c + e < a.vdim) o[c + e] = (__bf16)(x[e] * a.out_scale);
        }
    }
}

__global__ void __launch_bounds__(64) talk_merge_kernel(TalkArgs<__bf16> a) {
    const int row = blockIdx.x, h = blockIdx.y, used = used_splits(a, visible_keys(a, row));
    __bf16* o = a.out + (int64_t)row * a.out_row + (int64_t)h * a.vdim;
    for (int c = threadIdx.x * 4; c < a.vdim_pad; c += 256) {
        f32x4_t x = {0.f, 0.f, 0.f, 0.f};
        for (int s = 0; s < used; ++s)
            x += *reinterpret_cast<const f32x4_t*>(a.part + (((int64_t)row * a.splits + s) * a.heads + h) * a.vdim_pad + c);
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (c + e < a.vdim) o[c + e] = (__bf16)(x[e] * a.out_scale);
    }
}

// ------------------------------------------------------------------ launches
bool size_in(int64_t v, int64_t lo, int64_t hi) { return v >= lo && v <= hi; }

bool tiles_fit(int elem, int64_t heads, int64_t key_pad, int64_t vdim_pad, int64_t block_size) {
    return elem == INFER_ELEM_BF16 && heads <= 64 && key_pad <= 256 && vdim_pad <= 256 && block_size % kTile == 0;
}

template <class T>
int launch_any(const TalkArgs<T>& a, hipStream_t st) {
    const dim3 grid((unsigned)a.rows, (unsigned)a.heads), block(256);
    if (a.key_pad <= 128) hipLaunchKernelGGL((talk_scores_any_kernel<T, 2>), grid, block, 0, st, a);
    else if (a.key_pad <= 512) hipLaunchKernelGGL((talk_scores_any_kernel<T, 8>), grid, block, 0, st, a);
    else if (a.key_pad <= 1024) hipLaunchKernelGGL((talk_scores_any_kernel<T, 16>), grid, block, 0, st, a);
    else return INFER_KV_EUNSUPPORTED;
    int lanes = 16;
    while (lanes < 256 && lanes < a.vdim) lanes *= 2;
    const size_t lds = (size_t)(2 * a.heads + 512) * sizeof(float);
    if (a.vdim <= 256) hipLaunchKernelGGL((talk_values_any_kernel<T, 1>), grid, block, lds, st, a, lanes);
    else if (a.vdim <= 1024) hipLaunchKernelGGL((talk_values_any_kernel<T, 4>), grid, block, lds, st, a, lanes);
    else return INFER_KV_EUNSUPPORTED;
    return (int)hipGetLastError();
}

template <int MT, int KH, int NT>
int launch_values(const TalkArgs<__bf16>& a, dim3 grid, hipStream_t st) {
    const size_t lds = (size_t)kWaves * NT * 64 * sizeof(f32x4_t);     // the wavefronts' sums
    auto kernel = &talk_values_kernel<MT, KH, NT>;
    if (lds > 64 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return (int)e;
    }
    hipLaunchKernelGGL(kernel, grid, dim3(256), lds, st, a);
    return (int)hipGetLastError();
}

template <int MT>
int launch_tiles(TalkArgs<__bf16>& a, hipStream_t st) {
    const int shared = a.heads / a.kv_heads;
    a.groups = (unsigned)(a.kv_heads * ((shared + 16 * MT - 1) / (16 * MT)));
    const int64_t units = ((int64_t)a.rows * a.splits + 7) / 8 * 8;
    if (units * a.groups > 0x7fffffff) return INFER_KV_EINVAL;
    const dim3 grid((unsigned)(units * a.groups)), block(256);
    if (a.key_pad <= 64) hipLaunchKernelGGL((talk_scores_kernel<MT, 2>), grid, block, 0, st, a);
    else if (a.key_pad <= 128) hipLaunchKernelGGL((talk_scores_kernel<MT, 4>), grid, block, 0, st, a);
    else hipLaunchKernelGGL((talk_scores_kernel<MT, 8>), grid, block, 0, st, a);
    int rc = (int)hipGetLastError();
    if (rc) return rc;
    const bool one = a.heads <= 32;
    if (a.vdim_pad <= 64) rc = one ? launch_values<MT, 1, 4>(a, grid, st) : launch_values<MT, 2, 4>(a, grid, st);
    else if (a.vdim_pad <= 128) rc = one ? launch_values<MT, 1, 8>(a, grid, st) : launch_values<MT, 2, 8>(a, grid, st);
    else rc = one ? launch_values<MT, 1, 16>(a, grid, st) : launch_values<MT, 2, 16>(a, grid, st);
    if (rc || a.splits == 1) return rc;
    hipLaunchKernelGGL(talk_merge_kernel, dim3((unsigned)a.rows, (unsigned)a.heads), dim3(64), 0, st, a);
    return (int)hipGetLastError();
}

int64_t score_cap(int64_t max_keys) { return (max_keys + kTile - 1) / kTile * kTile; }

}  // namespace

extern "C" int64_t infer_talking_attention_splits(int elem, int64_t rows, int64_t heads, int64_t kv_heads, int64_t key_pad,
                                                  int64_t vdim_pad, int64_t block_size, int64_t max_keys) {
    if (!tiles_fit(elem, heads, key_pad, vdim_pad, block_size) || rows < 1 || heads < 1 || kv_heads < 1 || heads % kv_heads) return 1;
    const int64_t shared = heads / kv_heads, groups = kv_heads * (shared > 16 ? (shared + 31) / 32 : 1);
    int64_t splits = (1024 + rows * groups - 1) / (rows * groups);          // four workgroups per compute unit
    const int64_t most = (max_keys + 4 * kTile - 1) / (4 * kTile);          // a tile for every wavefront
    if (splits > most) splits = most;
    if (splits > 64) splits = 64;
    return splits < 1 ? 1 : splits;
}

extern "C" int64_t infer_talking_attention_workspace_floats(int64_t rows, int64_t heads, int64_t vdim_pad, int64_t splits, int64_t max_keys) {
    if (rows < 0 || heads < 1 || vdim_pad < 1 || splits < 1 || max_keys < 0) return 0;
    return rows * heads * (score_cap(max_keys) + splits * (2 + (splits > 1 ? vdim_pad : 0)));
}

extern "C" int infer_talking_attention(int elem, const void* qx, const void* keys, const void* values, int64_t key_pad, int64_t vdim_pad,
                                       const int32_t* block_table, int64_t bt_stride, int64_t table_cols, int64_t block_size,
                                       int64_t num_blocks, const int32_t* row_seq, const int32_t* ctx, int64_t rows, int64_t heads,
                                       int64_t kv_heads, float scale, const void* talk, float out_scale, int64_t splits, int64_t max_keys,
                                       void* out, int64_t out_stride, int64_t vdim, float* workspace, int64_t workspace_floats,
                                       void* stream) {
    if (!size_in(rows, 0, 0x7fffffff) || !size_in(kv_heads, 1, 4096) || !size_in(heads, 1, 4096) || heads % kv_heads ||
        !size_in(key_pad, 1, 1 << 16) || !size_in(vdim_pad, 1, 1 << 16) || !size_in(vdim, 1, vdim_pad) || !size_in(block_size, 1, 1 << 20) ||
        !size_in(table_cols, 1, 1 << 24) || table_cols * block_size > 0x7fffffff || num_blocks < 1 || bt_stride < table_cols ||
        out_stride < heads * vdim || !size_in(splits, 1, 64) || !size_in(max_keys, 1, 0x7fffffe0))
        return INFER_KV_EINVAL;
    if (rows == 0) return INFER_KV_OK;
    if (!qx || !keys || !values || !block_table || !ctx || !talk || !out) return INFER_KV_EINVAL;
    if (key_pad % 32 || vdim_pad % 32) return INFER_KV_EALIGN;
    if (!workspace || !ptr_aligned(workspace, 16) ||
        workspace_floats < infer_talking_attention_workspace_floats(rows, heads, vdim_pad, splits, max_keys))
        return INFER_KV_EWORKSPACE;
    hipStream_t st = (hipStream_t)stream;
    auto go = [&](auto zero) {
        using T = decltype(zero);
        const int64_t cap = score_cap(max_keys);
        float* part = workspace + rows * heads * cap;                       // 16-byte aligned, as are its rows
        TalkArgs<T> a{(const T*)qx, (const T*)keys, (const T*)values, (int)key_pad, (int)vdim_pad, block_table, bt_stride, (int)table_cols,
                      (int)block_size, (int)num_blocks, row_seq, ctx, (int)rows, (int)heads, (int)kv_heads, (int)splits, scale * kLog2e,
                      (const T*)talk, out_scale, (T*)out, out_stride, (int)vdim, workspace, cap,
                      part + (splits > 1 ? rows * splits * heads * vdim_pad : 0), part, 1};
        if constexpr (sizeof(T) == 2) {
            if (tiles_fit(elem, heads, key_pad, vdim_pad, block_size) && ptr_aligned(qx, 16) && ptr_aligned(keys, 16) && ptr_aligned(values, 16))
                return heads / kv_heads > 16 ? launch_tiles<2>(a, st) : launch_tiles<1>(a, st);
        }
        a.splits = 1;
        return launch_any(a, st);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}
