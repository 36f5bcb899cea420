// Latent attention over a paged cache of compressed rows, for gfx950 (MI355X).
//
// A cached token is one row shared by all heads: [ c (rank values, RMS-normed) | zeros | rotated key part | zeros ],
// both parts padded to 32 elements (`rank_pad`, `row` = rank_pad + padded rotated part).  Attention runs on
// these rows directly: the query is moved into the latent space (W_uk^T q per head), scores are dot products
// of whole rows, the weighted sum of the c parts is moved out again (W_uv per head).
//
//   latent_front_kernel     RMS norm of c, interleaved rotary on the shared key part and on the queries,
//                           append of the row to the cache
//   head_matmul_*           per-head products with W_uk^T and W_uv, the latter with the output gate
//   latent_rows_kernel      attention, any size and element type (one wavefront per key)
//   latent_decode_kernel    attention on MFMA tiles, keys split over workgroups, + latent_merge_kernel
//   latent_gather_kernel    cached rows of whole sequences as dense rows (for latent_prefill.hip)
//
// A query is a "row": a token, the block-table row of its sequence and the number of keys it sees.  A decode
// step has one row per sequence; the tokens of a short prompt portion are simply several rows.
#include "elem.h"

namespace {

typedef short i16x4 __attribute__((ext_vector_type(4)));
typedef short i16x8 __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) i16x4 lds_i16x4;

// ------------------------------------------------------------------ norm, rotary, append
template <class T>
struct LatentFrontArgs {
    T* proj; int64_t proj_stride;          // [q: heads x (dim + rot) | ... | c: rank, rotated part: rot | ...]
    int heads, dim, rot, rot_pairs, kv_off, rank;
    const float* c_norm; float eps;
    const float* table; int64_t max_pos;   // [max_pos][rot_pairs][cos, sin]
    const int64_t* positions;
    const int32_t* slots;
    T* cache; int rank_pad, row; int64_t num_slots;
    T* qx; int64_t qx_rows;                // rows below qx_rows: rotated q to qx[row][head][rank_pad ..], others in place
};

// a rotated pair in one access where every pair is aligned to its size (EVEN)
template <bool EVEN, class T>
__device__ __forceinline__ void load_pair(const T* p, float& u, float& v) {
    struct alignas(2 * sizeof(T)) Pair { T u, v; };
    if constexpr (EVEN) {
        const Pair x = *reinterpret_cast<const Pair*>(p);
        u = (float)x.u;
        v = (float)x.v;
    } else {
        u = (float)p[0];
        v = (float)p[1];
    }
}
template <bool EVEN, class T>
__device__ __forceinline__ void store_pair(T* p, float u, float v) {
    struct alignas(2 * sizeof(T)) Pair { T u, v; };
    if constexpr (EVEN) {
        *reinterpret_cast<Pair*>(p) = Pair{(T)u, (T)v};
    } else {
        p[0] = (T)u;
        p[1] = (T)v;
    }
}

template <class T, bool EVEN>
__global__ void __launch_bounds__(256) latent_front_kernel(LatentFrontArgs<T> a) {
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x;
    __shared__ float part[4];
    T* pr = a.proj + t * a.proj_stride;
    const T* kv = pr + a.kv_off;
    int64_t pos = a.positions[t];
    pos = pos < 0 ? 0 : (pos >= a.max_pos ? a.max_pos - 1 : pos);
    const float* cs = a.table + pos * (2 * a.rot_pairs);
    const int64_t slot = a.slots[t];

    float ss = 0.f;
    for (int r = tid; r < a.rank; r += 256) {
        const float v = (float)kv[r];
        ss += v * v;
    }
    const float rs = rsqrtf(block_sum<4>(ss, part) / (float)a.rank + a.eps);
    if (slot >= 0 && slot < a.num_slots) {
        T* row = a.cache + slot * a.row;
        for (int r = tid; r < a.rank_pad; r += 256) row[r] = r < a.rank ? (T)((float)kv[r] * rs * a.c_norm[r]) : (T)0.f;
        for (int i = tid; i < (a.row - a.rank_pad) / 2; i += 256) {
            float u = 0.f, v = 0.f;
            if (2 * i < a.rot) {
                load_pair<EVEN>(kv + a.rank + 2 * i, u, v);
                if (i < a.rot_pairs) {
                    const float c = cs[2 * i], s = cs[2 * i + 1];
                    const float u2 = u * c - v * s;
                    v = v * c + u * s;
                    u = u2;
                }
            }
            store_pair<EVEN>(row + a.rank_pad + 2 * i, u, v);
        }
    }
    const bool to_qx = t < a.qx_rows;
    const int pairs = to_qx ? (a.row - a.rank_pad) / 2 : a.rot / 2, total = a.heads * pairs;
    T* qx = to_qx ? a.qx + t * a.heads * a.row + a.rank_pad : pr + a.dim;
    const int qx_head = to_qx ? a.row : a.dim + a.rot;
    // four pairs per thread at a time, all loads in front of the stores
    for (int i0 = tid; i0 < total; i0 += 4 * 256) {
        float u[4], v[4], c[4], s[4];
        int h[4], p[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const int i = i0 + 256 * k < total ? i0 + 256 * k : i0;
            h[k] = i / pairs;
            p[k] = i - h[k] * pairs;
            u[k] = v[k] = s[k] = 0.f;
            c[k] = 1.f;
            if (2 * p[k] < a.rot) load_pair<EVEN>(pr + h[k] * (a.dim + a.rot) + a.dim + 2 * p[k], u[k], v[k]);
            if (p[k] < a.rot_pairs) { c[k] = cs[2 * p[k]]; s[k] = cs[2 * p[k] + 1]; }
        }
#pragma unroll
        for (int k = 0; k < 4; ++k)
            if (i0 + 256 * k < total) store_pair<EVEN>(qx + h[k] * qx_head + 2 * p[k], u[k] * c[k] - v[k] * s[k], v[k] * c[k] + u[k] * s[k]);
    }
}

// ------------------------------------------------------------------ per-head products
template <class T>
struct HeadMatmulArgs {
    const T* x; int64_t x_row, x_head;     // x[m][h][k]
    const T* w; int64_t w_head; int w_row; // w[h][n][k], k padded with zeros to w_row (a multiple of 32), n to 16
    T* out; int64_t out_row, out_head;     // out[m][h][n]
    const T* gate; int64_t gate_row;       // optional: out *= sigmoid(gate[m][h])
    int m, n, k;
};

template <class T>
__global__ void __launch_bounds__(256) head_matmul_any_kernel(HeadMatmulArgs<T> a) {
    extern __shared__ float xs[];
    const int m = blockIdx.x, h = blockIdx.y;
    const T* xr = a.x + (int64_t)m * a.x_row + (int64_t)h * a.x_head;
    for (int k = threadIdx.x; k < a.k; k += 256) xs[k] = (float)xr[k];
    __syncthreads();
    const float gate = a.gate ? sigmoid_f((float)a.gate[(int64_t)m * a.gate_row + h]) : 1.f;
    for (int n = threadIdx.x; n < a.n; n += 256) {
        const T* wr = a.w + (int64_t)h * a.w_head + (int64_t)n * a.w_row;
        float s = 0.f;
        for (int k = 0; k < a.k; ++k) s += xs[k] * (float)wr[k];
        a.out[(int64_t)m * a.out_row + (int64_t)h * a.out_head + n] = (T)(s * gate);
    }
}

// A wavefront owns 16 output columns of one head and up to MT x 16 rows: MFMA rows are the columns n (the
// weight, read once), MFMA columns the tokens.
template <int MT>
__global__ void __launch_bounds__(256) head_matmul_mfma_kernel(HeadMatmulArgs<__bf16> a) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int g = lane >> 4, c = lane & 15;
    const int n0 = (blockIdx.x * 4 + wave) * 16;
    if (n0 >= a.n) return;
    const int h = blockIdx.y, m0 = blockIdx.z * (16 * MT);
    const __bf16* wr = a.w + (int64_t)h * a.w_head + (int64_t)(n0 + c) * a.w_row + 8 * g;
    const __bf16* xr[MT];
    f32x4_t acc[MT];
#pragma unroll
    for (int u = 0; u < MT; ++u) {
        const int m = m0 + 16 * u + c;
        xr[u] = a.x + (int64_t)(m < a.m ? m : a.m - 1) * a.x_row + (int64_t)h * a.x_head + 8 * g;
        acc[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll 4
    for (int k = 0; k < a.k; k += 32) {
        const bf16x8_t w = *reinterpret_cast<const bf16x8_t*>(wr + k);
        const bool in = k + 8 * g < a.k;
#pragma unroll
        for (int u = 0; u < MT; ++u) {
            bf16x8_t x = {};
            if (in) x = *reinterpret_cast<const bf16x8_t*>(xr[u] + k);
            acc[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w, x, acc[u], 0, 0, 0);
        }
    }
#pragma unroll
    for (int u = 0; u < MT; ++u) {
        const int m = m0 + 16 * u + c;
        if (m >= a.m) continue;
        const float gate = a.gate ? sigmoid_f((float)a.gate[(int64_t)m * a.gate_row + h]) : 1.f;
        __bf16* o = a.out + (int64_t)m * a.out_row + (int64_t)h * a.out_head + n0 + 4 * g;
        if (n0 + 4 * g + 4 <= a.n) {
            bf16x4_t v;
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = (__bf16)(acc[u][e] * gate);
            *reinterpret_cast<bf16x4_t*>(o) = v;
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (n0 + 4 * g + e < a.n) o[e] = (__bf16)(acc[u][e] * gate);
        }
    }
}

// ------------------------------------------------------------------ attention over latent rows
template <class T>
struct LatentAttnArgs {
    const T* qx;                          // [rows][heads][row]
    const T* cache; int row, rank_pad;    // [blocks * block_size][row]
    const int32_t* bt; int64_t bt_stride; int table_cols, block_size, num_blocks;
    const int32_t* row_seq;               // block-table row of each query row; nullptr: the query row itself
    const int32_t* ctx;                   // keys each query row sees
    int heads, splits;
    float scale_log2;
    T* out;                               // [rows][heads][rank_pad]
    float* part;                          // [rows][splits][heads][rank_pad], then [rows][splits][heads][max, sum]
    float* part_ml;
    int rows; unsigned groups;            // MFMA kernel: query rows and head groups of the launch
};

template <class T>
__device__ __forceinline__ int visible_keys(const LatentAttnArgs<T>& a, int row) {
    const int len = a.ctx[row], cap = a.table_cols * a.block_size;
    return len < cap ? len : cap;         // a corrupt length cannot run past the table row
}
template <class T>
__device__ __forceinline__ int table_row(const LatentAttnArgs<T>& a, int row) {
    return a.row_seq ? a.row_seq[row] : row;
}
template <class T>
__device__ __forceinline__ int block_id(const LatentAttnArgs<T>& a, const int32_t* bt, int col) {
    const int b = bt[col];
    return b < 0 ? 0 : (b >= a.num_blocks ? a.num_blocks - 1 : b);
}

// One workgroup per (query row, head); wavefront w takes keys w, w + 4, ...; lanes hold the row elements
// lane, lane + 64, ...  NC = number of such elements a lane may hold.
template <class T, int NC>
__global__ void __launch_bounds__(256) latent_rows_kernel(LatentAttnArgs<T> a) {
    __shared__ float sm[4], sl[4];
    __shared__ float so[4][64 * NC];
    const int row = blockIdx.x, h = blockIdx.y;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int len = visible_keys(a, row);
    const int32_t* bt = a.bt + (int64_t)table_row(a, row) * a.bt_stride;
    const T* qr = a.qx + ((int64_t)row * a.heads + h) * a.row;
    float q[NC], o[NC];
#pragma unroll
    for (int i = 0; i < NC; ++i) {
        const int c = lane + 64 * i;
        q[i] = c < a.row ? (float)qr[c] * a.scale_log2 : 0.f;
        o[i] = 0.f;
    }
    float m = -INFINITY, l = 0.f;
    for (int key = wave; key < len; key += 4) {
        const int col = key / a.block_size;
        const T* kr = a.cache + ((int64_t)block_id(a, bt, col) * a.block_size + (key - col * a.block_size)) * a.row;
        float k[NC], s = 0.f;
#pragma unroll
        for (int i = 0; i < NC; ++i) {
            const int c = lane + 64 * i;
            k[i] = c < a.row ? (float)kr[c] : 0.f;
            s += q[i] * k[i];
        }
        s = wave_sum(s);
        const float mn = fmaxf(m, s);
        const float alpha = exp2f(m - mn), p = exp2f(s - mn);
        l = l * alpha + p;
#pragma unroll
        for (int i = 0; i < NC; ++i) o[i] = o[i] * alpha + p * k[i];
        m = mn;
    }
    if (lane == 0) { sm[wave] = m; sl[wave] = l; }
#pragma unroll
    for (int i = 0; i < NC; ++i) so[wave][lane + 64 * i] = o[i];
    __syncthreads();
    float mt = fmaxf(fmaxf(sm[0], sm[1]), fmaxf(sm[2], sm[3]));
    float w[4], lt = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        w[i] = sm[i] == -INFINITY ? 0.f : exp2f(sm[i] - mt);
        lt += sl[i] * w[i];
    }
    const float inv = lt > 0.f ? 1.f / lt : 0.f;
    T* out = a.out + ((int64_t)row * a.heads + h) * a.rank_pad;
    for (int c = threadIdx.x; c < a.rank_pad; c += 256) {
        float v = 0.f;
#pragma unroll
        for (int i = 0; i < 4; ++i) v += so[i][c] * w[i];
        out[c] = (T)(v * inv);
    }
}

// MFMA form.  A workgroup of four wavefronts serves MT x 16 heads of one query row over a run of 32-key tiles
// (split `blockIdx.x` of the keys).  A tile is contiguous in the cache (a block holds whole tiles), is staged
// through LDS once and serves both products:
//   S^T[key, head] = C[key, :] . Q^T     wavefront (key tile w % 2, half w / 2 of the k-steps), sums through LDS
//   O^T[c, head]  += C^T[c, key] . P^T   wavefront w owns the 16-channel tiles w, w + 4, ...
// The second product reads C transposed from LDS (ds_read_b64_tr_b16: lane i of a group of 16 points at 4
// consecutive elements of row i / 4 and receives column i of the 4 x 16 block).
constexpr int kTile = 32;
constexpr int kSRow = kTile + 4;      // floats per score row in LDS
constexpr float kLazy = 8.f;

__host__ __device__ constexpr int tile_pitch(int row) { return 2 * row + 16; }   // bytes: odd multiple of 16 modulo 256

template <int MT, int KSH, int NT>
__global__ void __launch_bounds__(256, 2) latent_decode_kernel(LatentAttnArgs<__bf16> a) {
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int g = lane >> 4, n = lane & 15;
    // Workgroups go to the eight dies round-robin: the head groups that read the same keys are given to one die, one
    // behind the other, so that its second-level cache serves all but the first of them.
    const unsigned die = blockIdx.x & 7u, turn = blockIdx.x >> 3;
    const unsigned unit = turn / a.groups * 8u + die;
    if (unit >= (unsigned)(a.rows * a.splits)) return;
    const int split = (int)(unit % (unsigned)a.splits), row = (int)(unit / (unsigned)a.splits);
    const int head0 = (int)(turn % a.groups) * (16 * MT);
    const int len = visible_keys(a, row);
    const int tiles = (len + kTile - 1) / kTile;
    const int per = (tiles + a.splits - 1) / a.splits;
    const int t0 = split * per, t1 = t0 + per < tiles ? t0 + per : tiles;
    if (t0 >= t1 && (a.splits > 1 || len > 0)) return;     // the merge knows which splits are empty
    const int32_t* bt = a.bt + (int64_t)table_row(a, row) * a.bt_stride;
    const int pitch = tile_pitch(a.row), ksteps = a.row / 32, ctiles = a.rank_pad / 16;
    float* sbuf = reinterpret_cast<float*>(lds + kTile * pitch);      // [2][MT * 16][kSRow]
    const int half = wave >> 1, ktile = wave & 1;

    bf16x8_t q[MT][KSH];
#pragma unroll
    for (int u = 0; u < MT; ++u) {
        const int h = head0 + 16 * u + n;
        const __bf16* qr = a.qx + ((int64_t)row * a.heads + (h < a.heads ? h : 0)) * a.row + 8 * g;
#pragma unroll
        for (int j = 0; j < KSH; ++j) {
            const int s = 2 * j + half;
            q[u][j] = bf16x8_t{};
            if (s < ksteps) q[u][j] = *reinterpret_cast<const bf16x8_t*>(qr + 32 * s);
        }
    }
    f32x4_t acc[MT][NT];
    float m[MT], l[MT];
#pragma unroll
    for (int u = 0; u < MT; ++u) {
        m[u] = -INFINITY;
        l[u] = 0.f;
#pragma unroll
        for (int i = 0; i < NT; ++i) acc[u][i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }

    // chunk i of this thread: 16 bytes at offset 16 (tid + 256 i) of the tile, and its place in LDS.  Sizes below what the
    // kernel is built for leave surplus chunks, which repeat the tile's last one (same bytes to the same place), surplus
    // k-steps, which meet zeros in q, and surplus channel tiles, which are not stored: no branches in the loop.
    const int chunks_per_row = a.row / 8, chunks = kTile * chunks_per_row;
    u32x4_t stage[KSH];
    int st_src[KSH], st_lds[KSH];
#pragma unroll
    for (int i = 0; i < KSH; ++i) {
        const int c = tid + 256 * i < chunks ? tid + 256 * i : chunks - 1;
        const int r = c / chunks_per_row;
        st_src[i] = 16 * c;
        st_lds[i] = r * pitch + (c - r * chunks_per_row) * 16;
    }
    int k_off[KSH];
#pragma unroll
    for (int j = 0; j < KSH; ++j) k_off[j] = __builtin_amdgcn_readfirstlane(2 * j + half < ksteps ? 64 * (2 * j + half) : 0);
    // tiles are walked in order: the block changes every `tiles_per_block` tiles, and its id is looked up a block ahead
    const int tiles_per_block = a.block_size / kTile;
    const int64_t tile_bytes = (int64_t)2 * kTile * a.row;
    int col = t0 / tiles_per_block, in_block = t0 - col * tiles_per_block;
    int next_id = block_id(a, bt, col);
    const unsigned char* src = nullptr;
    auto open_block = [&]() {
        src = reinterpret_cast<const unsigned char*>(a.cache) + ((int64_t)next_id * tiles_per_block + in_block) * tile_bytes;
        ++col;
        next_id = block_id(a, bt, col < a.table_cols ? col : a.table_cols - 1);
    };
    auto fetch = [&]() {
        if (in_block == tiles_per_block) {
            in_block = 0;
            open_block();
        }
#pragma unroll
        for (int i = 0; i < KSH; ++i) stage[i] = *reinterpret_cast<const u32x4_t*>(src + st_src[i]);
        src += tile_bytes;
        ++in_block;
    };
    if (t0 < t1) {
        open_block();
        fetch();
    }
    for (int t = t0; t < t1; ++t) {
        __syncthreads();
        if (len - t * kTile < kTile) {                            // rows behind the last key count as zeros
            const int have = 16 * (len - t * kTile) * chunks_per_row;
#pragma unroll
            for (int i = 0; i < KSH; ++i)
                if (st_src[i] >= have) stage[i] = u32x4_t{0u, 0u, 0u, 0u};
        }
#pragma unroll
        for (int i = 0; i < KSH; ++i) *reinterpret_cast<u32x4_t*>(lds + st_lds[i]) = stage[i];
        if (t + 1 < t1) fetch();
        __syncthreads();
        // ---- scores
        f32x4_t sc[MT];
#pragma unroll
        for (int u = 0; u < MT; ++u) sc[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        const unsigned char* kr = lds + (16 * ktile + n) * pitch + 16 * g;
#pragma unroll
        for (int j = 0; j < KSH; ++j) {
            const bf16x8_t kf = *reinterpret_cast<const bf16x8_t*>(kr + k_off[j]);
#pragma unroll
            for (int u = 0; u < MT; ++u) sc[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, q[u][j], sc[u], 0, 0, 0);
        }
#pragma unroll
        for (int u = 0; u < MT; ++u)
            *reinterpret_cast<f32x4_t*>(sbuf + (half * MT * 16 + 16 * u + n) * kSRow + 16 * ktile + 4 * g) = sc[u];
        __syncthreads();
        // ---- softmax over the 32 keys, in every wavefront: lane (g, n) has keys 8 g .. 8 g + 7 of head n.  The running
        // maximum moves only when it grows by more than kLazy (log2 units); until then weights are at most 2^kLazy.
        bf16x8_t pb[MT];
        const int seen = len - t * kTile - 8 * g;       // of this lane's keys the first `seen` exist
#pragma unroll
        for (int u = 0; u < MT; ++u) {
            const float* s0 = sbuf + (16 * u + n) * kSRow + 8 * g;
            const float* s1 = s0 + MT * 16 * kSRow;
            float sv[8];
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                const f32x4_t x = *reinterpret_cast<const f32x4_t*>(s0 + 4 * e), y = *reinterpret_cast<const f32x4_t*>(s1 + 4 * e);
#pragma unroll
                for (int i = 0; i < 4; ++i) sv[4 * e + i] = (x[i] + y[i]) * a.scale_log2;
            }
            if (len - t * kTile < kTile) {
#pragma unroll
                for (int i = 0; i < 8; ++i) sv[i] = i < seen ? sv[i] : -INFINITY;
            }
            float mx = sv[0];
#pragma unroll
            for (int i = 1; i < 8; ++i) mx = fmaxf(mx, sv[i]);
            mx = max_xor16_32(mx);
            const bool grow = mx > m[u] + kLazy;        // always in the first tile, whose first key exists
            if (__any(grow)) {
                const float alpha = grow ? __builtin_amdgcn_exp2f(m[u] - mx) : 1.f;
                m[u] = grow ? mx : m[u];
                l[u] *= alpha;
#pragma unroll
                for (int i = 0; i < NT; ++i) acc[u][i] *= alpha;
            }
            float sum = 0.f;
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const float p = __builtin_amdgcn_exp2f(sv[i] - m[u]);
                sum += p;
                pb[u][i] = (__bf16)p;
            }
            l[u] += sum;
        }
        // ---- weighted sum of the c parts
        const unsigned char* vr = lds + (8 * g + (n >> 2)) * pitch + (n & 3) * 8 + 32 * wave;
#pragma unroll
        for (int i = 0; i < NT; ++i) {
            const i16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(vr + 128 * i));
            const i16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(vr + 128 * i + 4 * pitch));
            const bf16x8_t vt = __builtin_bit_cast(bf16x8_t, (i16x8)__builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
#pragma unroll
            for (int u = 0; u < MT; ++u) acc[u][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, pb[u], acc[u][i], 0, 0, 0);
        }
    }
#pragma unroll
    for (int u = 0; u < MT; ++u) {
        const int h = head0 + 16 * u + n;
        float sum = l[u] + __shfl_xor(l[u], 16, 64);
        sum += __shfl_xor(sum, 32, 64);
        if (h >= a.heads) continue;
        if (a.splits == 1) {
            const float inv = sum > 0.f ? 1.f / sum : 0.f;
            __bf16* o = a.out + ((int64_t)row * a.heads + h) * a.rank_pad + 4 * g;
#pragma unroll
            for (int i = 0; i < NT; ++i) {
                const int ct = wave + 4 * i;
                if (ct < ctiles) {
                    bf16x4_t v;
#pragma unroll
                    for (int e = 0; e < 4; ++e) v[e] = (__bf16)(acc[u][i][e] * inv);
                    *reinterpret_cast<bf16x4_t*>(o + 16 * ct) = v;
                }
            }
        } else {
            const int64_t rec = ((int64_t)row * a.splits + split) * a.heads + h;
            float* o = a.part + rec * a.rank_pad + 4 * g;
#pragma unroll
            for (int i = 0; i < NT; ++i) {
                const int ct = wave + 4 * i;
                if (ct < ctiles) *reinterpret_cast<f32x4_t*>(o + 16 * ct) = acc[u][i];
            }
            if (wave == 0 && g == 0) { a.part_ml[2 * rec] = m[u]; a.part_ml[2 * rec + 1] = sum; }
        }
    }
}

__global__ void __launch_bounds__(128) latent_merge_kernel(LatentAttnArgs<__bf16> a) {
    const int row = blockIdx.x, h = blockIdx.y;
    const int tiles = (visible_keys(a, row) + kTile - 1) / kTile;
    const int per = (tiles + a.splits - 1) / a.splits;
    const int used = per > 0 ? (tiles + per - 1) / per : 0;
    const int64_t rec0 = (int64_t)row * a.splits * a.heads + h;
    float m = -INFINITY;
    for (int s = 0; s < used; ++s) m = fmaxf(m, a.part_ml[2 * (rec0 + (int64_t)s * a.heads)]);
    float l = 0.f;
    for (int s = 0; s < used; ++s) {
        const float* ml = a.part_ml + 2 * (rec0 + (int64_t)s * a.heads);
        l += ml[1] * exp2f(ml[0] - m);
    }
    const float inv = l > 0.f ? 1.f / l : 0.f;
    for (int c = threadIdx.x * 4; c < a.rank_pad; c += 512) {
        f32x4_t o = {0.f, 0.f, 0.f, 0.f};
        for (int s = 0; s < used; ++s) {
            const int64_t rec = rec0 + (int64_t)s * a.heads;
            o += *reinterpret_cast<const f32x4_t*>(a.part + rec * a.rank_pad + c) * exp2f(a.part_ml[2 * rec] - m);
        }
        bf16x4_t v;
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = (__bf16)(o[e] * inv);
        *reinterpret_cast<bf16x4_t*>(a.out + ((int64_t)row * a.heads + h) * a.rank_pad + c) = v;
    }
}

// ------------------------------------------------------------------ cached rows as dense rows
struct LatentGatherArgs {
    const uint16_t* cache; int row; int block_size, num_blocks, table_cols;
    const int32_t* bt; int64_t bt_stride;
    const int32_t* seqs;       // block-table row of each sequence
    const int32_t* cu_k;       // [sequences + 1] first dense row of each
    uint16_t* out;             // [total][row]
};

__global__ void __launch_bounds__(256) latent_gather_kernel(LatentGatherArgs a) {
    const int s = blockIdx.y;
    const int k0 = a.cu_k[s];
    int len = a.cu_k[s + 1] - k0;
    const int cap = a.table_cols * a.block_size;
    if (len > cap) len = cap;
    const int32_t* bt = a.bt + (int64_t)a.seqs[s] * a.bt_stride;
    const int chunks = a.row / 8;
    const int first = blockIdx.x * kTile;
    for (int i = threadIdx.x; i < kTile * chunks; i += 256) {
        const int t = first + i / chunks, c = i % chunks;
        if (t >= len) return;
        const int col = t / a.block_size;
        int b = bt[col];
        b = b < 0 ? 0 : (b >= a.num_blocks ? a.num_blocks - 1 : b);
        const u32x4_t v = *reinterpret_cast<const u32x4_t*>(a.cache + ((int64_t)b * a.block_size + (t - col * a.block_size)) * a.row + 8 * c);
        *reinterpret_cast<u32x4_t*>(a.out + (int64_t)(k0 + t) * a.row + 8 * c) = v;
    }
}

bool size_in(int64_t v, int64_t lo, int64_t hi) { return v >= lo && v <= hi; }

template <class T>
int launch_front(const LatentFrontArgs<T>& a, int64_t n, hipStream_t st) {
    const size_t pair = 2 * sizeof(T);
    const bool even = a.dim % 2 == 0 && a.rank % 2 == 0 && a.kv_off % 2 == 0 && a.proj_stride % 2 == 0 && ptr_aligned(a.proj, pair) &&
                      ptr_aligned(a.cache, pair) && ptr_aligned(a.qx, pair);
    if (even) hipLaunchKernelGGL((latent_front_kernel<T, true>), dim3((unsigned)n), dim3(256), 0, st, a);
    else hipLaunchKernelGGL((latent_front_kernel<T, false>), dim3((unsigned)n), dim3(256), 0, st, a);
    return (int)hipGetLastError();
}

template <class T>
int launch_rows(const LatentAttnArgs<T>& a, int64_t rows, hipStream_t st) {
    const dim3 grid((unsigned)rows, (unsigned)a.heads), block(256);
    if (a.row <= 128) hipLaunchKernelGGL((latent_rows_kernel<T, 2>), grid, block, 0, st, a);
    else if (a.row <= 256) hipLaunchKernelGGL((latent_rows_kernel<T, 4>), grid, block, 0, st, a);
    else if (a.row <= 640) hipLaunchKernelGGL((latent_rows_kernel<T, 10>), grid, block, 0, st, a);
    else if (a.row <= 1280) hipLaunchKernelGGL((latent_rows_kernel<T, 20>), grid, block, 0, st, a);
    else return INFER_KV_EUNSUPPORTED;
    return (int)hipGetLastError();
}

// sizes the MFMA attention kernel is built for
bool mfma_attention_fits(int64_t row, int64_t rank_pad, int64_t block_size) {
    return row <= 640 && rank_pad <= 512 && block_size % kTile == 0;
}

template <int KSH, int NT>
int launch_decode(LatentAttnArgs<__bf16>& a, hipStream_t st) {
    const int mt = a.heads > 16 ? 2 : 1;
    a.groups = (unsigned)((a.heads + 16 * mt - 1) / (16 * mt));
    const int64_t units = ((int64_t)a.rows * a.splits + 7) / 8 * 8;
    if (units * a.groups > 0x7fffffff) return INFER_KV_EINVAL;
    const dim3 grid((unsigned)(units * a.groups)), block(256);
    const size_t lds = (size_t)kTile * tile_pitch(a.row) + (size_t)2 * mt * 16 * kSRow * sizeof(float);
    if (mt == 2) hipLaunchKernelGGL((latent_decode_kernel<2, KSH, NT>), grid, block, lds, st, a);
    else hipLaunchKernelGGL((latent_decode_kernel<1, KSH, NT>), grid, block, lds, st, a);
    return (int)hipGetLastError();
}

}  // namespace

extern "C" int infer_latent_front(int elem, void* proj, int64_t proj_stride, int64_t heads, int64_t dim, int64_t rot,
                                  int64_t rot_dims, int64_t kv_off, int64_t rank, const float* c_norm, float eps,
                                  const float* table, int64_t max_pos, const int64_t* positions, const int32_t* slots,
                                  void* cache, int64_t rank_pad, int64_t row, int64_t num_slots, void* qx,
                                  int64_t qx_rows, int64_t n, void* stream) {
    if (n < 0 || n > 0x7fffffff) return INFER_KV_EINVAL;
    if (n == 0) return INFER_KV_OK;
    if (!proj || !c_norm || !table || !positions || !slots || !cache || (qx_rows > 0 && !qx)) return INFER_KV_EINVAL;
    if (!size_in(heads, 1, 4096) || !size_in(dim, 1, 65536) || !size_in(rot, 2, 65536) || rot % 2 || rot_dims % 2 ||
        rot_dims < 0 || rot_dims > rot || !size_in(rank, 1, rank_pad) || !size_in(rank_pad + rot, 1, row) ||
        row > (1 << 20) || rank_pad % 2 || row % 2 || max_pos < 1 || num_slots < 1 || qx_rows < 0 || qx_rows > n)
        return INFER_KV_EINVAL;
    if (kv_off < heads * (dim + rot) || proj_stride < kv_off + rank + rot) return INFER_KV_EINVAL;
    if (elem == INFER_ELEM_BF16) {
        LatentFrontArgs<__bf16> a{(__bf16*)proj, proj_stride, (int)heads, (int)dim, (int)rot, (int)(rot_dims / 2), (int)kv_off,
                                  (int)rank, c_norm, eps, table, max_pos, positions, slots, (__bf16*)cache, (int)rank_pad,
                                  (int)row, num_slots, (__bf16*)qx, qx_rows};
        return launch_front(a, n, (hipStream_t)stream);
    }
    if (elem == INFER_ELEM_F32) {
        LatentFrontArgs<float> a{(float*)proj, proj_stride, (int)heads, (int)dim, (int)rot, (int)(rot_dims / 2), (int)kv_off,
                                 (int)rank, c_norm, eps, table, max_pos, positions, slots, (float*)cache, (int)rank_pad,
                                 (int)row, num_slots, (float*)qx, qx_rows};
        return launch_front(a, n, (hipStream_t)stream);
    }
    return INFER_KV_EUNSUPPORTED;
}

extern "C" int infer_head_matmul(int elem, const void* x, int64_t x_row, int64_t x_head, const void* w, int64_t w_head,
                                 int64_t w_row, void* out, int64_t out_row, int64_t out_head, const void* gate,
                                 int64_t gate_row, int64_t m, int64_t heads, int64_t n, int64_t k, void* stream) {
    if (m < 0 || m > 0x7fffffff) return INFER_KV_EINVAL;
    if (m == 0) return INFER_KV_OK;
    if (!x || !w || !out || !size_in(heads, 1, 4096) || !size_in(n, 1, 1 << 20) || !size_in(k, 1, 16384)) return INFER_KV_EINVAL;
    if (w_row < k || w_row % 32 || w_head < (n + 15) / 16 * 16 * w_row || (gate && gate_row < heads)) return INFER_KV_EINVAL;
    hipStream_t st = (hipStream_t)stream;
    if (elem == INFER_ELEM_BF16) {
        HeadMatmulArgs<__bf16> a{(const __bf16*)x, x_row, x_head, (const __bf16*)w, w_head, (int)w_row, (__bf16*)out, out_row,
                                 out_head, (const __bf16*)gate, gate_row, (int)m, (int)n, (int)k};
        const bool tiles = k % 8 == 0 && x_row % 8 == 0 && x_head % 8 == 0 && out_row % 4 == 0 && out_head % 4 == 0 &&
                           ptr_aligned(x, 16) && ptr_aligned(w, 16) && ptr_aligned(out, 8);
        if (tiles) {
            const unsigned gx = (unsigned)((n + 63) / 64);
            // few workgroups: 16 rows each instead of 64, the weights then come from the second-level cache
            if (m <= 16 || (m + 63) / 64 * gx * heads < 512) {
                hipLaunchKernelGGL((head_matmul_mfma_kernel<1>), dim3(gx, (unsigned)heads, (unsigned)((m + 15) / 16)), dim3(256), 0, st, a);
            } else {
                if ((m + 63) / 64 > 65535) return INFER_KV_EINVAL;
                hipLaunchKernelGGL((head_matmul_mfma_kernel<4>), dim3(gx, (unsigned)heads, (unsigned)((m + 63) / 64)), dim3(256), 0, st, a);
            }
            return (int)hipGetLastError();
        }
        hipLaunchKernelGGL((head_matmul_any_kernel<__bf16>), dim3((unsigned)m, (unsigned)heads), dim3(256), k * sizeof(float), st, a);
        return (int)hipGetLastError();
    }
    if (elem == INFER_ELEM_F32) {
        HeadMatmulArgs<float> a{(const float*)x, x_row, x_head, (const float*)w, w_head, (int)w_row, (float*)out, out_row,
                                out_head, (const float*)gate, gate_row, (int)m, (int)n, (int)k};
        hipLaunchKernelGGL((head_matmul_any_kernel<float>), dim3((unsigned)m, (unsigned)heads), dim3(256), k * sizeof(float), st, a);
        return (int)hipGetLastError();
    }
    return INFER_KV_EUNSUPPORTED;
}

extern "C" int64_t infer_latent_attention_splits(int elem, int64_t rows, int64_t heads, int64_t row, int64_t rank_pad,
                                                 int64_t block_size, int64_t max_keys) {
    if (elem != INFER_ELEM_BF16 || !mfma_attention_fits(row, rank_pad, block_size) || rows < 1 || heads < 1) return 1;
    // two workgroups are resident per compute unit; more splits than that only add partial results
    const int64_t groups = heads > 16 ? (heads + 31) / 32 : 1;
    int64_t splits = (512 + rows * groups - 1) / (rows * groups);
    const int64_t most = (max_keys + 4 * kTile - 1) / (4 * kTile);     // no split shorter than four tiles
    if (splits > most) splits = most;
    if (splits > 64) splits = 64;
    return splits < 1 ? 1 : splits;
}

extern "C" int infer_latent_attention(int elem, const void* qx, const void* cache, int64_t row, int64_t rank_pad,
                                      const int32_t* block_table, int64_t bt_stride, int64_t table_cols, int64_t block_size,
                                      int64_t num_blocks, const int32_t* row_seq, const int32_t* ctx, int64_t rows,
                                      int64_t heads, float scale, int64_t splits, void* out, float* workspace,
                                      int64_t workspace_floats, void* stream) {
    if (rows < 0 || rows > 0x7fffffff) return INFER_KV_EINVAL;
    if (rows == 0) return INFER_KV_OK;
    if (!qx || !cache || !block_table || !ctx || !out) return INFER_KV_EINVAL;
    if (!size_in(heads, 1, 4096) || !size_in(row, 1, 1 << 20) || !size_in(rank_pad, 1, row) || !size_in(block_size, 1, 1 << 20) ||
        !size_in(table_cols, 1, 1 << 24) || table_cols * block_size > 0x7fffffff || num_blocks < 1 || bt_stride < table_cols)
        return INFER_KV_EINVAL;
    if (row % 32 || rank_pad % 32) return INFER_KV_EALIGN;
    if (!size_in(splits, 1, 64)) return INFER_KV_EINVAL;
    hipStream_t st = (hipStream_t)stream;
    const float scale_log2 = scale * kLog2e;
    if (elem == INFER_ELEM_F32) {
        LatentAttnArgs<float> a{(const float*)qx, (const float*)cache, (int)row, (int)rank_pad, block_table, bt_stride, (int)table_cols,
                                (int)block_size, (int)num_blocks, row_seq, ctx, (int)heads, 1, scale_log2, (float*)out, nullptr, nullptr, (int)rows, 1};
        return launch_rows(a, rows, st);
    }
    if (elem != INFER_ELEM_BF16) return INFER_KV_EUNSUPPORTED;
    LatentAttnArgs<__bf16> a{(const __bf16*)qx, (const __bf16*)cache, (int)row, (int)rank_pad, block_table, bt_stride, (int)table_cols,
                             (int)block_size, (int)num_blocks, row_seq, ctx, (int)heads, (int)splits, scale_log2, (__bf16*)out,
                             workspace, workspace ? workspace + rows * splits * heads * rank_pad : nullptr, (int)rows, 1};
    if (!mfma_attention_fits(row, rank_pad, block_size) || !ptr_aligned(qx, 16) || !ptr_aligned(cache, 16) || !ptr_aligned(out, 8)) {
        a.splits = 1;
        return launch_rows(a, rows, st);
    }
    if (splits > 1 && (!workspace || !ptr_aligned(workspace, 16) || workspace_floats < rows * splits * heads * (rank_pad + 2)))
        return INFER_KV_EWORKSPACE;
    int rc;
    if (row <= 192 && rank_pad <= 128) rc = launch_decode<3, 2>(a, st);
    else if (row <= 384 && rank_pad <= 256) rc = launch_decode<6, 4>(a, st);
    else if (row <= 576) rc = launch_decode<9, 8>(a, st);
    else rc = launch_decode<10, 8>(a, st);
    if (rc) return rc;
    if (splits > 1) hipLaunchKernelGGL(latent_merge_kernel, dim3((unsigned)rows, (unsigned)heads), dim3(128), 0, st, a);
    return (int)hipGetLastError();
}

extern "C" int infer_latent_gather(const void* cache, int64_t row, int64_t block_size, int64_t num_blocks,
                                   const int32_t* block_table, int64_t bt_stride, int64_t table_cols, const int32_t* seqs,
                                   const int32_t* cu_k, int64_t num_seqs, int64_t max_keys, void* out, void* stream) {
    if (num_seqs < 0 || max_keys < 0 || num_seqs > 65535) return INFER_KV_EINVAL;
    if (num_seqs == 0 || max_keys == 0) return INFER_KV_OK;
    if (!cache || !block_table || !seqs || !cu_k || !out || row <= 0 || row > (1 << 20) || block_size <= 0 || num_blocks <= 0 ||
        table_cols <= 0 || table_cols * block_size > 0x7fffffff || bt_stride < table_cols)
        return INFER_KV_EINVAL;
    if (row % 8 || !ptr_aligned(cache, 16) || !ptr_aligned(out, 16)) return INFER_KV_EALIGN;
    LatentGatherArgs a{(const uint16_t*)cache, (int)row, (int)block_size, (int)num_blocks, (int)table_cols, block_table, bt_stride,
                       seqs, cu_k, (uint16_t*)out};
    hipLaunchKernelGGL(latent_gather_kernel, dim3((unsigned)((max_keys + kTile - 1) / kTile), (unsigned)num_seqs), dim3(256), 0,
                       (hipStream_t)stream, a);
    return (int)hipGetLastError();
}
