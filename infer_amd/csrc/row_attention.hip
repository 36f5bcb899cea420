// Attention of query rows over paged rows, for gfx950 (MI355X).
//
// A query is a "row": a token, the block-table row of its sequence and the number of keys it sees.  A decode step has
// one row per sequence; the tokens of a short prompt portion are simply several rows.  A cached row holds values in
// front and the key: the two overlap in latent attention (the whole row is the key, its first part the value), and
// stand one behind the other in grouped attention, which has a row per token and key/value head.
//
//   row_attention_any_kernel     any size and element type (one wavefront per key)
//   row_attention_tile_kernel    MFMA tiles, keys split over workgroups, + row_attention_merge_kernel
//   row_gather_kernel            cached rows of whole sequences as dense rows (for dense_prefill.hip)
//
// The softmax may have a sink (a learned score per head with neither key nor value), the scores a bias that grows with the
// distance, the output a gate per head.  A query may see only the keys of its chunk or of a window (masks.h).
//
// A head may have two maps: two attentions over the same values whose difference is the output.  Each map is a query head
// of its own here (its query is zero where the other map's key stands in the row), their sums stay unreduced, and
//   row_attention_merge2_kernel  takes the difference, norms it and applies the gate.
#include "elem.h"
#include "masks.h"

namespace {

typedef short i16x4 __attribute__((ext_vector_type(4)));
typedef short i16x8 __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) i16x4 lds_i16x4;

template <class T>
struct RowAttnArgs {
    const T* qx;                          // [rows][heads][key_len]
    const T* cache; int row;              // [blocks][kv_heads][block_size][row]
    int val_len, key_off, key_len;        // a row's values: [0, val_len), its key: [key_off, key_off + key_len)
    const int32_t* bt; int64_t bt_stride; int table_cols, block_size, num_blocks;
    const int32_t* row_seq;               // block-table row of each query row; nullptr: the query row itself
    const int32_t* ctx;                   // keys each query row sees
    int heads, kv_heads, splits;          // heads / kv_heads consecutive query heads share a row
    float scale_log2;
    const float* sink;                    // [heads] or nullptr: a score of its own in the denominator
    const T* gate; int64_t gate_row;      // optional: out *= sigmoid(gate[query row][head])
    T* out; int64_t out_row; int out_head, out_n;   // [rows][heads][out_n]: the first out_n values
    bool out_vec;                         // four values may be stored at once
    float* part;                          // [rows][splits][heads][val_len], then [rows][splits][heads][max, sum]
    float* part_ml;
    int rows; unsigned groups;            // MFMA kernel: query rows and head groups of the launch
    KeyMask mask;                         // which of the keys in front of it a query sees
    bool biased;                          // scores lose distance_slope(head) per token of distance
    float out_scale;                      // of the output
    bool keep_parts;                      // two maps: sums are left in part, part_ml
};

template <class T>
__device__ __forceinline__ int visible_keys(const RowAttnArgs<T>& a, int row) {
    const int len = a.ctx[row], cap = a.table_cols * a.block_size;
    return len < cap ? len : cap;         // a corrupt length cannot run past the table row
}
template <class T>
__device__ __forceinline__ int table_row(const RowAttnArgs<T>& a, int row) {
    return a.row_seq ? a.row_seq[row] : row;
}
template <class T>
__device__ __forceinline__ int block_id(const RowAttnArgs<T>& a, const int32_t* bt, int col) {
    const int b = bt[col];
    return b < 0 ? 0 : (b >= a.num_blocks ? a.num_blocks - 1 : b);
}

// What a head's weighted sum is multiplied by: one over the softmax denominator (`sum` relative to 2^m, the sink
// beside it, counted here and nowhere else), and the output gate.
template <class T>
__device__ __forceinline__ float out_factor(const RowAttnArgs<T>& a, int row, int h, float m, float sum) {
    if (a.sink && sum > 0.f) sum += exp2f(a.sink[h] * kLog2e - m);
    const float inv = sum > 0.f ? a.out_scale / sum : 0.f;
    return a.gate ? inv * sigmoid_f((float)a.gate[(int64_t)row * a.gate_row + h]) : inv;
}
template <class T>
__device__ __forceinline__ T* out_row(const RowAttnArgs<T>& a, int row, int h) {
    return a.out + (int64_t)row * a.out_row + (int64_t)h * a.out_head;
}
// values c .. c + 3 of a head
__device__ __forceinline__ void store_values(const RowAttnArgs<__bf16>& a, __bf16* o, int c, f32x4_t x) {
    bf16x4_t v;
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = (__bf16)x[e];
    if (a.out_vec && c + 4 <= a.out_n) {
        *reinterpret_cast<bf16x4_t*>(o + c) = v;
    } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (c + e < a.out_n) o[c + e] = v[e];
    }
}

// One workgroup per (query row, head); wavefront w takes keys w, w + 4, ...; lanes hold the row elements
// lane, lane + 64, ...  NC = number of such elements a lane may hold.
template <class T, int NC>
__global__ void __launch_bounds__(256) row_attention_any_kernel(RowAttnArgs<T> a) {
    __shared__ float sm[4], sl[4];
    __shared__ float so[4][64 * NC];
    const int row = blockIdx.x, h = blockIdx.y;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int len = visible_keys(a, row);
    const int32_t* bt = a.bt + (int64_t)table_row(a, row) * a.bt_stride;
    const int kvh = h / (a.heads / a.kv_heads);
    const T* qr = a.qx + ((int64_t)row * a.heads + h) * a.key_len - a.key_off;
    float q[NC], o[NC];
#pragma unroll
    for (int i = 0; i < NC; ++i) {
        const int c = lane + 64 * i;
        q[i] = c >= a.key_off && c < a.key_off + a.key_len ? (float)qr[c] * a.scale_log2 : 0.f;
        o[i] = 0.f;
    }
    float m = -INFINITY, l = 0.f;
    const float slope = a.biased ? distance_slope(h, a.heads) * kLog2e : 0.f;
    for (int key = a.mask.first(len - 1) + wave; key < len; key += 4) {
        const int col = key / a.block_size;
        const T* kr = a.cache + (((int64_t)block_id(a, bt, col) * a.kv_heads + kvh) * a.block_size + (key - col * a.block_size)) * a.row;
        float k[NC], s = 0.f;
#pragma unroll
        for (int i = 0; i < NC; ++i) {
            const int c = lane + 64 * i;
            k[i] = c < a.row ? (float)kr[c] : 0.f;
            s += q[i] * k[i];
        }
        s = wave_sum(s) - slope * (float)(len - 1 - key);
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
    const int64_t rec = (int64_t)row * a.heads + h;
    const float f = a.keep_parts ? 1.f : out_factor(a, row, h, mt, lt);
    T* out = a.keep_parts ? nullptr : out_row(a, row, h);
    for (int c = threadIdx.x; c < (a.keep_parts ? a.val_len : a.out_n); c += 256) {
        float v = 0.f;
#pragma unroll
        for (int i = 0; i < 4; ++i) v += so[i][c] * w[i];
        if (a.keep_parts) a.part[rec * a.val_len + c] = v;
        else out[c] = (T)(v * f);
    }
    if (a.keep_parts && threadIdx.x == 0) {
        a.part_ml[2 * rec] = mt;
        a.part_ml[2 * rec + 1] = lt;
    }
}

// MFMA form.  A workgroup of four wavefronts serves MT x 16 heads (of one key/value head) of one query row over a run of 32-key tiles
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

template <int MT, int KSH, int NT, int SH>
__global__ void __launch_bounds__(256, 2) row_attention_tile_kernel(RowAttnArgs<__bf16> a) {
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
    const int shared = a.heads / a.kv_heads, per_kv = (shared + 16 * MT - 1) / (16 * MT);
    const int kvh = (int)(turn % a.groups) / per_kv;
    const int head0 = kvh * shared + ((int)(turn % a.groups) - kvh * per_kv) * (16 * MT), head_end = (kvh + 1) * shared;
    const int len = visible_keys(a, row);
    const int lo = a.mask.first(len - 1), tiles = (len + kTile - 1) / kTile, tile0 = lo / kTile;
    const int per = (tiles - tile0 + a.splits - 1) / a.splits;
    const int t0 = tile0 + split * per, t1 = t0 + per < tiles ? t0 + per : tiles;
    if (t0 >= t1 && (a.splits > 1 || len > 0)) return;     // the merge knows which splits are empty
    const int32_t* bt = a.bt + (int64_t)table_row(a, row) * a.bt_stride;
    const int pitch = tile_pitch(a.row), ksteps = a.key_len / 32, ctiles = a.val_len / 16;
    float* sbuf = reinterpret_cast<float*>(lds + kTile * pitch);      // [2][MT * 16][kSRow]
    const int half = wave >> 1, ktile = wave & 1;

    bf16x8_t q[MT][KSH];
#pragma unroll
    for (int u = 0; u < MT; ++u) {
        const int h = head0 + 16 * u + n;
        const __bf16* qr = a.qx + ((int64_t)row * a.heads + (h < head_end ? h : head0)) * a.key_len + 8 * g;
#pragma unroll
        for (int j = 0; j < KSH; ++j) {
            const int s = 2 * j + half;
            q[u][j] = bf16x8_t{};
            if (s < ksteps) q[u][j] = *reinterpret_cast<const bf16x8_t*>(qr + 32 * s);
        }
    }
    f32x4_t acc[MT][NT];
    float m[MT], l[MT], slope[MT];
#pragma unroll
    for (int u = 0; u < MT; ++u) {
        m[u] = -INFINITY;
        l[u] = 0.f;
        slope[u] = a.biased ? distance_slope(head0 + 16 * u + n, a.heads) * kLog2e : 0.f;
#pragma unroll
        for (int i = 0; i < NT; ++i) acc[u][i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }

    // chunk i of this thread: 16 bytes at offset 16 (tid + 256 i) of the tile, and its place in LDS.  Sizes below what the
    // kernel is built for leave surplus chunks, which repeat the tile's last one (same bytes to the same place), surplus
    // k-steps, which meet zeros in q, and surplus channel tiles, which are not stored: no branches in the loop.
    const int chunks_per_row = a.row / 8, chunks = kTile * chunks_per_row;
    u32x4_t stage[SH];
    int st_src[SH], st_lds[SH];
#pragma unroll
    for (int i = 0; i < SH; ++i) {
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
        src = reinterpret_cast<const unsigned char*>(a.cache) + (((int64_t)next_id * a.kv_heads + kvh) * tiles_per_block + in_block) * tile_bytes;
        ++col;
        next_id = block_id(a, bt, col < a.table_cols ? col : a.table_cols - 1);
    };
    auto fetch = [&]() {
        if (in_block == tiles_per_block) {
            in_block = 0;
            open_block();
        }
#pragma unroll
        for (int i = 0; i < SH; ++i) stage[i] = *reinterpret_cast<const u32x4_t*>(src + st_src[i]);
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
            for (int i = 0; i < SH; ++i)
                if (st_src[i] >= have) stage[i] = u32x4_t{0u, 0u, 0u, 0u};
        }
#pragma unroll
        for (int i = 0; i < SH; ++i) *reinterpret_cast<u32x4_t*>(lds + st_lds[i]) = stage[i];
        if (t + 1 < t1) fetch();
        __syncthreads();
        // ---- scores
        f32x4_t sc[MT];
#pragma unroll
        for (int u = 0; u < MT; ++u) sc[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        const unsigned char* kr = lds + (16 * ktile + n) * pitch + 2 * a.key_off + 16 * g;
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
        const int hidden = lo - t * kTile - 8 * g;      // and the first `hidden` lie in front of what the query sees
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
            if (a.biased) {
#pragma unroll
                for (int i = 0; i < 8; ++i) sv[i] += slope[u] * (float)(i + 1 - seen);
            }
            if (len - t * kTile < kTile || t == tile0) {
#pragma unroll
                for (int i = 0; i < 8; ++i) sv[i] = i < seen && i >= hidden ? sv[i] : -INFINITY;
            }
            float mx = sv[0];
#pragma unroll
            for (int i = 1; i < 8; ++i) mx = fmaxf(mx, sv[i]);
            mx = max_xor16_32(mx);
            const bool grow = mx > m[u] + kLazy;        // always in the first tile, which has a key that is seen
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
        // ---- weighted sum of the values
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
        if (h >= head_end) continue;
        if (a.splits == 1 && !a.keep_parts) {
            const float f = out_factor(a, row, h, m[u], sum);
            __bf16* o = out_row(a, row, h);
#pragma unroll
            for (int i = 0; i < NT; ++i) {
                const int ct = wave + 4 * i;
                if (ct < ctiles) store_values(a, o, 16 * ct + 4 * g, acc[u][i] * f);
            }
        } else {
            const int64_t rec = ((int64_t)row * a.splits + split) * a.heads + h;
            float* o = a.part + rec * a.val_len + 4 * g;
#pragma unroll
            for (int i = 0; i < NT; ++i) {
                const int ct = wave + 4 * i;
                if (ct < ctiles) *reinterpret_cast<f32x4_t*>(o + 16 * ct) = acc[u][i];
            }
            if (wave == 0 && g == 0) { a.part_ml[2 * rec] = m[u]; a.part_ml[2 * rec + 1] = sum; }
        }
    }
}

// splits of a query row that have keys
template <class T>
__device__ __forceinline__ int used_splits(const RowAttnArgs<T>& a, int row) {
    const int len = visible_keys(a, row), tiles = (len + kTile - 1) / kTile - a.mask.first(len - 1) / kTile;
    const int per = (tiles + a.splits - 1) / a.splits;
    return per > 0 ? (tiles + per - 1) / per : 0;
}

// Two maps: out = rms(o1 - lambda o2) * gain, with the gate.  One wavefront per (query row, head).
struct TwoMaps { float lambda, gain, eps; };
template <class T, int NC>
__global__ void __launch_bounds__(64) row_attention_merge2_kernel(RowAttnArgs<T> a, TwoMaps d) {
    const int row = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
    const int used = used_splits(a, row);
    float o[NC];
#pragma unroll
    for (int i = 0; i < NC; ++i) o[i] = 0.f;
#pragma unroll
    for (int map = 0; map < 2; ++map) {
        const int64_t rec0 = (int64_t)row * a.splits * a.heads + 2 * h + map;
        float m = -INFINITY, l = 0.f;
        for (int s = 0; s < used; ++s) m = fmaxf(m, a.part_ml[2 * (rec0 + (int64_t)s * a.heads)]);
        for (int s = 0; s < used; ++s) {
            const float* ml = a.part_ml + 2 * (rec0 + (int64_t)s * a.heads);
            l += ml[1] * exp2f(ml[0] - m);
        }
        const float f = l > 0.f ? (map ? -d.lambda : 1.f) / l : 0.f;
        for (int s = 0; s < used; ++s) {
            const int64_t rec = rec0 + (int64_t)s * a.heads;
            const float w = f * exp2f(a.part_ml[2 * rec] - m);
#pragma unroll
            for (int i = 0; i < NC; ++i)
                if (lane + 64 * i < a.out_n) o[i] += w * a.part[rec * a.val_len + lane + 64 * i];
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NC; ++i) ss += o[i] * o[i];
    float f = rsqrtf(wave_sum(ss) / (float)a.out_n + d.eps) * d.gain;
    if (a.gate) f *= sigmoid_f((float)a.gate[(int64_t)row * a.gate_row + h]);
    T* out = out_row(a, row, h);
#pragma unroll
    for (int i = 0; i < NC; ++i)
        if (lane + 64 * i < a.out_n) out[lane + 64 * i] = (T)(o[i] * f);
}

__global__ void __launch_bounds__(128) row_attention_merge_kernel(RowAttnArgs<__bf16> a) {
    const int row = blockIdx.x, h = blockIdx.y;
    const int used = used_splits(a, row);
    const int64_t rec0 = (int64_t)row * a.splits * a.heads + h;
    float m = -INFINITY;
    for (int s = 0; s < used; ++s) m = fmaxf(m, a.part_ml[2 * (rec0 + (int64_t)s * a.heads)]);
    float l = 0.f;
    for (int s = 0; s < used; ++s) {
        const float* ml = a.part_ml + 2 * (rec0 + (int64_t)s * a.heads);
        l += ml[1] * exp2f(ml[0] - m);
    }
    const float f = out_factor(a, row, h, m, l);
    __bf16* out = out_row(a, row, h);
    for (int c = threadIdx.x * 4; c < a.val_len; c += 512) {
        f32x4_t o = {0.f, 0.f, 0.f, 0.f};
        for (int s = 0; s < used; ++s) {
            const int64_t rec = rec0 + (int64_t)s * a.heads;
            o += *reinterpret_cast<const f32x4_t*>(a.part + rec * a.val_len + c) * exp2f(a.part_ml[2 * rec] - m);
        }
        store_values(a, out, c, o * f);
    }
}

// ------------------------------------------------------------------ cached rows as dense rows
struct RowGatherArgs {
    const uint16_t* cache; int row, kv_heads; int block_size, num_blocks, table_cols;
    const int32_t* bt; int64_t bt_stride;
    const int32_t* seqs;       // block-table row of each sequence
    const int32_t* cu_k;       // [sequences + 1] first dense row of each
    uint16_t* out;             // [total][kv_heads][row]
    const int32_t* cu_q;       // [sequences + 1] or nullptr: rows that no query of these portions sees are left out
    KeyMask mask;
};

__global__ void __launch_bounds__(256) row_gather_kernel(RowGatherArgs a) {
    const int s = blockIdx.y;
    const int k0 = a.cu_k[s];
    int len = a.cu_k[s + 1] - k0;
    const int cap = a.table_cols * a.block_size;
    if (len > cap) len = cap;
    const int32_t* bt = a.bt + (int64_t)a.seqs[s] * a.bt_stride;
    const int row_chunks = a.row / 8, chunks = a.kv_heads * row_chunks;
    const int first = blockIdx.x * kTile;
    if (a.cu_q && first + kTile <= a.mask.first(len - (a.cu_q[s + 1] - a.cu_q[s])) / kTile * kTile) return;
    for (int i = threadIdx.x; i < kTile * chunks; i += 256) {
        const int t = first + i / chunks, c = i % chunks;
        if (t >= len) return;
        const int col = t / a.block_size;
        int b = bt[col];
        b = b < 0 ? 0 : (b >= a.num_blocks ? a.num_blocks - 1 : b);
        const int h = c / row_chunks;
        const u32x4_t v = *reinterpret_cast<const u32x4_t*>(
            a.cache + (((int64_t)b * a.kv_heads + h) * a.block_size + (t - col * a.block_size)) * a.row + 8 * (c - h * row_chunks));
        *reinterpret_cast<u32x4_t*>(a.out + ((int64_t)(k0 + t) * chunks + c) * 8) = v;
    }
}

template <class T>
int launch_any(const RowAttnArgs<T>& a, int64_t rows, hipStream_t st) {
    const dim3 grid((unsigned)rows, (unsigned)a.heads), block(256);
    if (a.row <= 128) hipLaunchKernelGGL((row_attention_any_kernel<T, 2>), grid, block, 0, st, a);
    else if (a.row <= 256) hipLaunchKernelGGL((row_attention_any_kernel<T, 4>), grid, block, 0, st, a);
    else if (a.row <= 640) hipLaunchKernelGGL((row_attention_any_kernel<T, 10>), grid, block, 0, st, a);
    else if (a.row <= 1280) hipLaunchKernelGGL((row_attention_any_kernel<T, 20>), grid, block, 0, st, a);
    else return INFER_KV_EUNSUPPORTED;
    return (int)hipGetLastError();
}

// sizes the MFMA attention kernel is built for
bool tiles_fit(int64_t row, int64_t val_len, int64_t block_size) {
    return row <= 640 && val_len <= 512 && block_size % kTile == 0;
}

template <int KSH, int NT, int SH>
int launch_tiles(RowAttnArgs<__bf16>& a, hipStream_t st) {
    const int shared = a.heads / a.kv_heads, mt = shared > 16 ? 2 : 1;
    a.groups = (unsigned)(a.kv_heads * ((shared + 16 * mt - 1) / (16 * mt)));
    const int64_t units = ((int64_t)a.rows * a.splits + 7) / 8 * 8;
    if (units * a.groups > 0x7fffffff) return INFER_KV_EINVAL;
    const dim3 grid((unsigned)(units * a.groups)), block(256);
    const size_t lds = (size_t)kTile * tile_pitch(a.row) + (size_t)2 * mt * 16 * kSRow * sizeof(float);
    if (mt == 2) hipLaunchKernelGGL((row_attention_tile_kernel<2, KSH, NT, SH>), grid, block, lds, st, a);
    else hipLaunchKernelGGL((row_attention_tile_kernel<1, KSH, NT, SH>), grid, block, lds, st, a);
    return (int)hipGetLastError();
}

bool size_in(int64_t v, int64_t lo, int64_t hi) { return v >= lo && v <= hi; }

int64_t row_splits(int elem, int64_t rows, int64_t heads, int64_t kv_heads, int64_t row, int64_t val_len, int64_t block_size,
                   int64_t max_keys, int64_t resident) {
    if (elem != INFER_ELEM_BF16 || !tiles_fit(row, val_len, block_size) || rows < 1 || heads < 1 || kv_heads < 1 || heads % kv_heads) return 1;
    // as many workgroups as are resident; more splits than that only add partial results
    const int64_t shared = heads / kv_heads, groups = kv_heads * (shared > 16 ? (shared + 31) / 32 : 1);
    int64_t splits = (resident + rows * groups - 1) / (rows * groups);
    const int64_t most = (max_keys + 4 * kTile - 1) / (4 * kTile);     // no split shorter than four tiles
    if (splits > most) splits = most;
    if (splits > 64) splits = 64;
    return splits < 1 ? 1 : splits;
}

// checks what both forms of attention share and runs the kernels; `a` has everything but the workspace
template <class T>
int run_rows(RowAttnArgs<T>& a, float* workspace, int64_t workspace_floats, hipStream_t st) {
    if (a.rows == 0) return INFER_KV_OK;
    if (!a.qx || !a.cache || !a.bt || !a.ctx || !a.out) return INFER_KV_EINVAL;
    if (!size_in(a.splits, 1, 64)) return INFER_KV_EINVAL;
    const bool tiled = sizeof(T) == 2 && tiles_fit(a.row, a.val_len, a.block_size) && ptr_aligned(a.qx, 16) && ptr_aligned(a.cache, 16);
    if (!tiled) a.splits = 1;
    const int64_t records = (int64_t)a.rows * a.splits * a.heads;
    if constexpr (sizeof(T) == 2) {
        if (!tiled) goto any;
        if (a.splits > 1 || a.keep_parts) {
            if (!workspace || !ptr_aligned(workspace, 16) || workspace_floats < records * (a.val_len + 2)) return INFER_KV_EWORKSPACE;
            a.part = workspace;
            a.part_ml = workspace + records * a.val_len;
        }
        int rc;
        if (a.key_off == 0) {                                    // values and key overlap
            if (a.row <= 192 && a.val_len <= 128) rc = launch_tiles<3, 2, 3>(a, st);
            else if (a.row <= 384 && a.val_len <= 256) rc = launch_tiles<6, 4, 6>(a, st);
            else if (a.row <= 576) rc = launch_tiles<9, 8, 9>(a, st);
            else rc = launch_tiles<10, 8, 10>(a, st);
        } else if (a.key_len <= 64 && a.val_len <= 64) rc = launch_tiles<1, 1, 2>(a, st);
        else if (a.key_len <= 128 && a.val_len <= 128) rc = launch_tiles<2, 2, 4>(a, st);
        else if (a.key_len <= 256 && a.val_len <= 256) rc = launch_tiles<4, 4, 8>(a, st);
        else rc = launch_tiles<10, 8, 10>(a, st);
        if (rc) return rc;
        if (a.splits > 1 && !a.keep_parts) hipLaunchKernelGGL(row_attention_merge_kernel, dim3((unsigned)a.rows, (unsigned)a.heads), dim3(128), 0, st, a);
        return (int)hipGetLastError();
    }
any:
    if (a.keep_parts) {
        if (!workspace || !ptr_aligned(workspace, 16) || workspace_floats < records * (a.val_len + 2)) return INFER_KV_EWORKSPACE;
        a.part = workspace;
        a.part_ml = workspace + records * a.val_len;
    }
    return launch_any(a, a.rows, st);
}

// both maps' sums, then their difference; `a` has the maps as query heads
template <class T>
int run_two_maps(RowAttnArgs<T>& a, TwoMaps d, float* workspace, int64_t workspace_floats, hipStream_t st) {
    a.keep_parts = true;
    if (a.rows == 0) return INFER_KV_OK;
    if (a.out_n > 1024) return INFER_KV_EUNSUPPORTED;
    const int rc = run_rows(a, workspace, workspace_floats, st);
    if (rc) return rc;
    const dim3 grid((unsigned)a.rows, (unsigned)(a.heads / 2)), block(64);
    if (a.out_n <= 64) hipLaunchKernelGGL((row_attention_merge2_kernel<T, 1>), grid, block, 0, st, a, d);
    else if (a.out_n <= 128) hipLaunchKernelGGL((row_attention_merge2_kernel<T, 2>), grid, block, 0, st, a, d);
    else if (a.out_n <= 256) hipLaunchKernelGGL((row_attention_merge2_kernel<T, 4>), grid, block, 0, st, a, d);
    else hipLaunchKernelGGL((row_attention_merge2_kernel<T, 16>), grid, block, 0, st, a, d);
    return (int)hipGetLastError();
}

int row_gather(const void* cache, int64_t row, int64_t kv_heads, int64_t block_size, int64_t num_blocks, const int32_t* block_table,
               int64_t bt_stride, int64_t table_cols, const int32_t* seqs, const int32_t* cu_k, int64_t num_seqs, int64_t max_keys,
               void* out, void* stream, const int32_t* cu_q = nullptr, KeyMask mask = KeyMask{}) {
    if (num_seqs < 0 || max_keys < 0 || num_seqs > 65535) return INFER_KV_EINVAL;
    if (num_seqs == 0 || max_keys == 0) return INFER_KV_OK;
    if (!cache || !block_table || !seqs || !cu_k || !out || row <= 0 || row > (1 << 20) || kv_heads < 1 || kv_heads > 4096 ||
        block_size <= 0 || num_blocks <= 0 || table_cols <= 0 || table_cols * block_size > 0x7fffffff || bt_stride < table_cols)
        return INFER_KV_EINVAL;
    if (row % 8 || !ptr_aligned(cache, 16) || !ptr_aligned(out, 16)) return INFER_KV_EALIGN;
    RowGatherArgs a{(const uint16_t*)cache, (int)row, (int)kv_heads, (int)block_size, (int)num_blocks, (int)table_cols, block_table,
                    bt_stride, seqs, cu_k, (uint16_t*)out, cu_q, mask};
    hipLaunchKernelGGL(row_gather_kernel, dim3((unsigned)((max_keys + kTile - 1) / kTile), (unsigned)num_seqs), dim3(256), 0,
                       (hipStream_t)stream, a);
    return (int)hipGetLastError();
}

}  // namespace

extern "C" int64_t infer_latent_attention_splits(int elem, int64_t rows, int64_t heads, int64_t row, int64_t rank_pad,
                                                 int64_t block_size, int64_t max_keys) {
    return row_splits(elem, rows, heads, 1, row, rank_pad, block_size, max_keys, 512);     // two per compute unit
}

extern "C" int infer_latent_attention(int elem, const void* qx, const void* cache, int64_t row, int64_t rank_pad,
                                      const int32_t* block_table, int64_t bt_stride, int64_t table_cols, int64_t block_size,
                                      int64_t num_blocks, const int32_t* row_seq, const int32_t* ctx, int64_t rows,
                                      int64_t heads, float scale, int64_t splits, void* out, float* workspace,
                                      int64_t workspace_floats, void* stream) {
    if (!size_in(rows, 0, 0x7fffffff) || !size_in(heads, 1, 4096) || !size_in(row, 1, 1 << 20) || !size_in(rank_pad, 1, row) ||
        !size_in(block_size, 1, 1 << 20) || !size_in(table_cols, 1, 1 << 24) || table_cols * block_size > 0x7fffffff ||
        num_blocks < 1 || bt_stride < table_cols)
        return INFER_KV_EINVAL;
    if (row % 32 || rank_pad % 32) return INFER_KV_EALIGN;
    auto go = [&](auto zero) {
        using T = decltype(zero);
        RowAttnArgs<T> a{(const T*)qx, (const T*)cache, (int)row, (int)rank_pad, 0, (int)row, block_table, bt_stride, (int)table_cols,
                         (int)block_size, (int)num_blocks, row_seq, ctx, (int)heads, 1, (int)splits, scale * kLog2e, nullptr, nullptr, 0,
                         (T*)out, heads * rank_pad, (int)rank_pad, (int)rank_pad, ptr_aligned(out, 8), nullptr, nullptr, (int)rows, 1,
                         KeyMask{}, false, 1.f, false};
        return run_rows(a, workspace, workspace_floats, (hipStream_t)stream);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}

extern "C" int infer_latent_gather(const void* cache, int64_t row, int64_t block_size, int64_t num_blocks,
                                   const int32_t* block_table, int64_t bt_stride, int64_t table_cols, const int32_t* seqs,
                                   const int32_t* cu_k, int64_t num_seqs, int64_t max_keys, void* out, void* stream) {
    return row_gather(cache, row, 1, block_size, num_blocks, block_table, bt_stride, table_cols, seqs, cu_k, num_seqs, max_keys, out, stream);
}

extern "C" int64_t infer_grouped_attention_splits(int elem, int64_t rows, int64_t heads, int64_t kv_heads, int64_t dim_pad,
                                                  int64_t vdim_pad, int64_t block_size, int64_t max_keys) {
    return row_splits(elem, rows, heads, kv_heads, dim_pad + vdim_pad, vdim_pad, block_size, max_keys, 1024);
}

extern "C" int infer_grouped_attention(int elem, const void* qx, const void* cache, int64_t dim_pad, int64_t vdim_pad,
                                       const int32_t* block_table, int64_t bt_stride, int64_t table_cols, int64_t block_size,
                                       int64_t num_blocks, const int32_t* row_seq, const int32_t* ctx, int64_t rows,
                                       int64_t heads, int64_t kv_heads, float scale, const float* sink, const void* gate,
                                       int64_t gate_stride, int64_t splits, void* out, int64_t out_stride, int64_t vdim,
                                       float* workspace, int64_t workspace_floats, void* stream) {
    if (!size_in(rows, 0, 0x7fffffff) || !size_in(kv_heads, 1, 4096) || !size_in(heads, 1, 4096) || heads % kv_heads ||
        !size_in(dim_pad, 1, 1 << 16) || !size_in(vdim_pad, 1, 1 << 16) || !size_in(vdim, 1, vdim_pad) ||
        !size_in(block_size, 1, 1 << 20) || !size_in(table_cols, 1, 1 << 24) || table_cols * block_size > 0x7fffffff ||
        num_blocks < 1 || bt_stride < table_cols || out_stride < heads * vdim || (gate && gate_stride < heads))
        return INFER_KV_EINVAL;
    if (dim_pad % 32 || vdim_pad % 32) return INFER_KV_EALIGN;
    auto go = [&](auto zero) {
        using T = decltype(zero);
        RowAttnArgs<T> a{(const T*)qx, (const T*)cache, (int)(dim_pad + vdim_pad), (int)vdim_pad, (int)vdim_pad, (int)dim_pad, block_table,
                         bt_stride, (int)table_cols, (int)block_size, (int)num_blocks, row_seq, ctx, (int)heads, (int)kv_heads,
                         (int)splits, scale * kLog2e, sink, (const T*)gate, gate_stride, (T*)out, out_stride, (int)vdim, (int)vdim,
                         ptr_aligned(out, 4 * sizeof(T)) && out_stride % 4 == 0 && vdim % 4 == 0, nullptr, nullptr, (int)rows, 1,
                         KeyMask{}, false, 1.f, false};
        return run_rows(a, workspace, workspace_floats, (hipStream_t)stream);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}

extern "C" int infer_grouped_gather(const void* cache, int64_t row, int64_t kv_heads, int64_t block_size, int64_t num_blocks,
                                    const int32_t* block_table, int64_t bt_stride, int64_t table_cols, const int32_t* seqs,
                                    const int32_t* cu_k, int64_t num_seqs, int64_t max_keys, void* out, void* stream) {
    return row_gather(cache, row, kv_heads, block_size, num_blocks, block_table, bt_stride, table_cols, seqs, cu_k, num_seqs, max_keys,
                      out, stream);
}

extern "C" int infer_masked_attention(int elem, const void* qx, const void* cache, int64_t key_pad, int64_t vdim_pad,
                                      const int32_t* block_table, int64_t bt_stride, int64_t table_cols, int64_t block_size,
                                      int64_t num_blocks, const int32_t* row_seq, const int32_t* ctx, int64_t rows, int64_t heads,
                                      int64_t kv_heads, int64_t maps, float scale, int mask_kind, int64_t mask_size, int biased,
                                      const float* sink, const void* gate, int64_t gate_stride, float out_scale, float lambda,
                                      float eps, int64_t splits, void* out, int64_t out_stride, int64_t vdim, float* workspace,
                                      int64_t workspace_floats, void* stream) {
    if (!size_in(rows, 0, 0x7fffffff) || !size_in(kv_heads, 1, 4096) || !size_in(heads, 1, 4096) || heads % kv_heads ||
        !size_in(maps, 1, 2) || !size_in(key_pad, 1, 1 << 16) || !size_in(vdim_pad, 1, 1 << 16) || !size_in(vdim, 1, vdim_pad) ||
        !size_in(block_size, 1, 1 << 20) || !size_in(table_cols, 1, 1 << 24) || table_cols * block_size > 0x7fffffff ||
        num_blocks < 1 || bt_stride < table_cols || out_stride < heads * vdim || (gate && gate_stride < heads) ||
        (maps == 2 && (sink || biased)) || !mask_valid(mask_kind, mask_size))
        return INFER_KV_EINVAL;
    if (key_pad % 32 || vdim_pad % 32) return INFER_KV_EALIGN;
    auto go = [&](auto zero) {
        using T = decltype(zero);
        RowAttnArgs<T> a{(const T*)qx, (const T*)cache, (int)(key_pad + vdim_pad), (int)vdim_pad, (int)vdim_pad, (int)key_pad, block_table,
                         bt_stride, (int)table_cols, (int)block_size, (int)num_blocks, row_seq, ctx, (int)(heads * maps), (int)kv_heads,
                         (int)splits, scale * kLog2e, sink, (const T*)gate, gate_stride, (T*)out, out_stride, (int)vdim, (int)vdim,
                         ptr_aligned(out, 4 * sizeof(T)) && out_stride % 4 == 0 && vdim % 4 == 0, nullptr, nullptr, (int)rows, 1,
                         KeyMask{mask_kind, (int)mask_size}, biased != 0, out_scale, false};
        if (maps == 2) return run_two_maps(a, TwoMaps{lambda, out_scale, eps}, workspace, workspace_floats, (hipStream_t)stream);
        return run_rows(a, workspace, workspace_floats, (hipStream_t)stream);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}

extern "C" int infer_masked_gather(const void* cache, int64_t row, int64_t kv_heads, int64_t block_size, int64_t num_blocks,
                                   const int32_t* block_table, int64_t bt_stride, int64_t table_cols, const int32_t* seqs,
                                   const int32_t* cu_q, const int32_t* cu_k, int64_t num_seqs, int64_t max_keys, int mask_kind,
                                   int64_t mask_size, void* out, void* stream) {
    if (!cu_q || !mask_valid(mask_kind, mask_size)) return INFER_KV_EINVAL;
    return row_gather(cache, row, kv_heads, block_size, num_blocks, block_table, bt_stride, table_cols, seqs, cu_k, num_seqs, max_keys,
                      out, stream, cu_q, KeyMask{mask_kind, (int)mask_size});
}
