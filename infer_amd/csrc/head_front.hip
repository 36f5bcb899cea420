// Front end of attention with heads of their own norms, for gfx950 (MI355X): per token the biases of the projections, an RMS norm over
// every head's query and key (with or without a weight) and over its value (without), rotary positions (entry i turns with entry
// i + half), a factor of the query that grows with the position, and the append of one key and one value per key/value head: to
// pages of [value | key] rows (row_attention.hip) or to pages of tiles (tile_pages.h).
//
// A head may have two maps: two queries and two keys beside one value.  Each map is a vector of its own here.  The cached
// row is [value | key of map 1 | key of map 2], and a query that goes to the row kernels is padded to the length of both keys,
// with zeros where the other map's key stands.
#include "elem.h"
#include "tile_pages.h"

namespace {

template <class T>
struct HeadFrontArgs {
    T* proj; int64_t proj_stride; int q_off, k_off, v_off;   // heads x maps x dim, kv_heads x maps x dim, kv_heads x vdim
    int heads, kv_heads, maps, dim, vdim, half;              // half: rotated pairs
    const float* bias;                     // per column of proj, or nullptr
    const float* q_norm; const float* k_norm; float eps;     // [dim], nullptr: no weight
    bool norm_qk, norm_v;
    float temp_coef; double temp_every;    // q *= 1 + temp_coef ln(floor((position + 1) / temp_every) + 1), 0: no factor
    const float* table; int64_t max_pos;   // [max_pos][half][cos, sin]
    const int64_t* positions;
    const int32_t* slots;
    T* keys; T* values; int key_row, value_row;              // [blocks][kv_heads][block_size][..]: elements per token
    bool tiles;                                              // tile_pages.h, or a token's entries one behind the other
    bool apart;                                              // fill_tiles_kernel has keys and values
    int block_size, key_pad, vdim_pad; int64_t num_slots;
    T* qx; int64_t qx_rows;                // rows below qx_rows: q to qx[row][head][map][key_pad], others in place
};

template <class T, int N>
__device__ __forceinline__ void load_biased(const HeadFrontArgs<T>& a, const T* pr, int col, float (&x)[N]) {
    load_elems<N>(pr + col, x);
    if (a.bias) {
        float b[N];
        load_elems<N>(a.bias + col, b);
#pragma unroll
        for (int e = 0; e < N; ++e) x[e] += b[e];
    }
}

// where a token's key and value of key/value head 0 go, nullptr if it has no place; the next head's is block_size rows on
template <class T>
struct Slot { T* key; T* value; int64_t key_head, value_head; };
template <class T>
__device__ __forceinline__ Slot<T> slot_of(const HeadFrontArgs<T>& a, int64_t slot) {
    const int64_t kh = (int64_t)a.block_size * a.key_row, vh = (int64_t)a.block_size * a.value_row;
    if (slot < 0 || slot >= a.num_slots) return {nullptr, nullptr, kh, vh};
    const int64_t block = slot / a.block_size;
    const int off = (int)(slot - block * a.block_size), in_tile = a.tiles ? off % kTileTokens : 0;
    const int64_t row = block * a.kv_heads * a.block_size + off - in_tile;
    return {a.keys + row * a.key_row + tile_key_entry(in_tile, 0), a.values + row * a.value_row + tile_value_entry(in_tile, 0), kh, vh};
}

// where vector i (queries first, then keys, then values unless they are copied as they are) of a token comes from and goes to; to == nullptr: nowhere
template <class T>
struct Place {
    int from, size; T* to; const float* weight; bool norm, rotated; float factor;
    bool key_tile, value_tile;
    __device__ __forceinline__ T* at(int d) const { return to + (key_tile ? tile_key_entry(0, d) : value_tile ? tile_value_entry(0, d) : d); }
    __device__ __forceinline__ void store(int d, const float (&x)[8]) const {
        if (!value_tile) {
            store_elems<8>(at(d), x);                        // eight entries are neighbours in a tile, too
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) *at(d + e) = (T)x[e];
        }
    }
};
template <class T>
__device__ __forceinline__ Place<T> place_of(const HeadFrontArgs<T>& a, T* pr, const Slot<T>& s, T* qx, float factor, int i) {
    const int nq = a.heads * a.maps, nk = a.kv_heads * a.maps;
    if (i < nq) {
        const int from = a.q_off + i * a.dim;
        return {from, a.dim, qx ? qx + (int64_t)i * a.key_pad + i % a.maps * a.dim : pr + from, a.q_norm, a.norm_qk, true, factor, false, false};
    }
    i -= nq;
    if (i < nk) return {a.k_off + i * a.dim, a.dim, s.key ? s.key + i / a.maps * s.key_head + i % a.maps * a.dim : nullptr, a.k_norm, a.norm_qk, true, 1.f, a.tiles, false};
    i -= nk;
    return {a.v_off + i * a.vdim, a.vdim, s.value ? s.value + i * s.value_head : nullptr, nullptr, a.norm_v, false, 1.f, false, a.tiles};
}
template <class T>
__host__ __device__ __forceinline__ int num_vectors(const HeadFrontArgs<T>& a) {
    return (a.heads + (a.apart ? 0 : a.kv_heads)) * a.maps + ((a.norm_v || a.tiles) && !a.apart ? a.kv_heads : 0);
}

template <class T>
__device__ __forceinline__ float query_factor(const HeadFrontArgs<T>& a, int64_t pos) {
    return a.temp_every > 0.0 ? 1.f + a.temp_coef * logf((float)(floor((double)(pos + 1) / a.temp_every) + 1.0)) : 1.f;
}

// values that are stored as they are
template <class T, int N>
__device__ __forceinline__ void copy_values(const HeadFrontArgs<T>& a, const T* pr, const Slot<T>& s) {
    if (!s.value || a.norm_v || a.tiles) return;
    for (int i = threadIdx.x; i < a.kv_heads * a.vdim / N; i += 256) {
        float v[N];
        load_biased(a, pr, a.v_off + N * i, v);
        const int h = N * i / a.vdim;
        store_elems<N>(s.value + h * s.value_head + (N * i - h * a.vdim), v);
    }
}

// zeros that the attention kernels read: behind the real sizes, and at the other map's place in a query
template <class T>
__device__ __forceinline__ void fill_padding(const HeadFrontArgs<T>& a, const Slot<T>& s, T* qx) {
    const int used = a.maps * a.dim, pad = a.key_pad - used, vpad = a.vdim_pad - a.vdim;
    if (s.key && !a.apart) {
        for (int i = threadIdx.x; i < a.kv_heads * pad; i += 256) {
            const int d = used + i % pad;
            s.key[i / pad * s.key_head + (a.tiles ? tile_key_entry(0, d) : d)] = (T)0.f;
        }
        for (int i = threadIdx.x; i < a.kv_heads * vpad; i += 256) {
            const int d = a.vdim + i % vpad;
            s.value[i / vpad * s.value_head + (a.tiles ? tile_value_entry(0, d) : d)] = (T)0.f;
        }
    }
    if (qx) {
        const int rest = a.key_pad - a.dim;
        for (int i = threadIdx.x; i < a.heads * a.maps * rest; i += 256) {
            const int v = i / rest, c = i % rest, own = v % a.maps * a.dim;
            qx[(int64_t)v * a.key_pad + (c < own ? c : c + a.dim)] = (T)0.f;
        }
    }
}

// LANES lanes per vector, eight entries each; NV vectors per thread; sizes, offsets and the number of pairs are multiples of
// eight.  A vector lies in one wavefront, so its entries are all read before any is written in place.
template <class T, int LANES, int NV>
__global__ void __launch_bounds__(256) head_front_kernel(HeadFrontArgs<T> a) {
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x, c = 8 * (tid % LANES);
    T* pr = a.proj + t * a.proj_stride;
    const Slot<T> slot = slot_of(a, a.slots[t]);
    T* qx = t < a.qx_rows ? a.qx + t * a.heads * a.maps * a.key_pad : nullptr;
    const int total = num_vectors(a);
    int64_t pos = a.positions[t] < 0 ? 0 : a.positions[t];
    const float factor = query_factor(a, pos);
    pos = pos >= a.max_pos ? a.max_pos - 1 : pos;
    const bool low = c < a.half, turned = c < 2 * a.half;
    float x[NV][8];
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int i = tid / LANES + j * (256 / LANES);
#pragma unroll
        for (int e = 0; e < 8; ++e) x[j][e] = 0.f;
        const Place<T> p = place_of(a, pr, slot, qx, factor, i < total ? i : 0);
        if (c < p.size && i < total) load_biased(a, pr, p.from + c, x[j]);
    }
    float turn[16];
    if (turned) {
        const float* cs = a.table + (pos * a.half + (low ? c : c - a.half)) * 2;
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const f32x4_t v = reinterpret_cast<const f32x4_t*>(cs)[k];
#pragma unroll
            for (int e = 0; e < 4; ++e) turn[4 * k + e] = v[e];
        }
    }
    copy_values<T, 8>(a, pr, slot);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int i = tid / LANES + j * (256 / LANES);
        const Place<T> p = place_of(a, pr, slot, qx, factor, i < total ? i : 0);
        const bool in = c < p.size;
        if (a.norm_qk || a.norm_v) {                              // entries behind the size are zero
            float s = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) s += x[j][e] * x[j][e];
#pragma unroll
            for (int m = LANES / 2; m >= 1; m >>= 1) s += __shfl_xor(s, m, 64);
            if (p.norm) {
                const float r = rsqrtf(s / (float)p.size + a.eps);
                float w[8];
#pragma unroll
                for (int e = 0; e < 8; ++e) w[e] = 1.f;
                if (in && p.weight) load_elems<8>(p.weight + c, w);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[j][e] *= r * w[e];
            }
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) x[j][e] *= p.factor;
        if (a.half > 0) {
            const int other = (tid & 63) + (low ? a.half / 8 : turned ? -(a.half / 8) : 0);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float y = __shfl(x[j][e], other, 64);
                if (turned && p.rotated) x[j][e] = x[j][e] * turn[2 * e] + (low ? -y : y) * turn[2 * e + 1];
            }
        }
        if (in && i < total && p.to) p.store(c, x[j]);
    }
    fill_padding(a, slot, qx);
}

// any size: one wavefront per vector
template <class T>
__global__ void __launch_bounds__(256) head_front_any_kernel(HeadFrontArgs<T> a) {
    const int64_t t = blockIdx.x;
    const int lane = threadIdx.x & 63;
    T* pr = a.proj + t * a.proj_stride;
    const Slot<T> slot = slot_of(a, a.slots[t]);
    T* qx = t < a.qx_rows ? a.qx + t * a.heads * a.maps * a.key_pad : nullptr;
    int64_t pos = a.positions[t] < 0 ? 0 : a.positions[t];
    const float factor = query_factor(a, pos);
    pos = pos >= a.max_pos ? a.max_pos - 1 : pos;
    const float* cs = a.table + pos * (2 * a.half);
    for (int i = threadIdx.x >> 6; i < num_vectors(a); i += 4) {
        const Place<T> p = place_of(a, pr, slot, qx, factor, i);
        float r = p.factor;
        if (p.norm) {
            float s = 0.f, x[1];
            for (int d = lane; d < p.size; d += 64) {
                load_biased(a, pr, p.from + d, x);
                s += x[0] * x[0];
            }
            r *= rsqrtf(wave_sum(s) / (float)p.size + a.eps);
        }
        if (!p.to) continue;
        // a pair is read and written by one lane
        const int half = p.rotated ? a.half : 0;
        for (int d = lane; d < p.size - half; d += 64) {
            const bool pair = d < half;
            const int at = pair ? d : d + half;
            float u[1], v[1] = {0.f};
            load_biased(a, pr, p.from + at, u);
            u[0] *= p.weight ? r * p.weight[at] : r;
            if (pair) {
                load_biased(a, pr, p.from + d + a.half, v);
                v[0] *= p.weight ? r * p.weight[d + a.half] : r;
                const float co = cs[2 * d], si = cs[2 * d + 1];
                *p.at(d + a.half) = (T)(v[0] * co + u[0] * si);
                u[0] = u[0] * co - v[0] * si;
            }
            *p.at(at) = (T)u[0];
        }
    }
    copy_values<T, 1>(a, pr, slot);
    fill_padding(a, slot, qx);
}

// Keys or values of one head of 32 consecutive tokens to tiles, with neighbouring tokens in one store or in neighbouring lanes.  No biases,
// rotation or second map.  Eight threads per token, NC chunks of eight entries each.  blockIdx.y: heads of keys, then of values.
template <class T, int NC>
__global__ void __launch_bounds__(256) fill_tiles_kernel(HeadFrontArgs<T> a, int64_t n) {
    constexpr int kRow = 64 * NC + 8;                            // entries of a token in LDS
    __shared__ __attribute__((aligned(16))) T tile[32 * kRow];
    __shared__ int64_t slot[32];
    const int64_t t0 = (int64_t)blockIdx.x * 32;
    const bool is_key = (int)blockIdx.y < a.kv_heads, norm = is_key ? a.norm_qk : a.norm_v;
    const int tid = threadIdx.x, r = tid / 8, h = is_key ? blockIdx.y : blockIdx.y - a.kv_heads;
    const int size = is_key ? a.dim : a.vdim, pad = is_key ? a.key_pad : a.vdim_pad;
    const T* pr = a.proj + (t0 + r < n ? t0 + r : t0) * a.proj_stride + (is_key ? a.k_off : a.v_off) + h * size;
    if (tid < 32) {
        const int64_t s = t0 + tid < n ? a.slots[t0 + tid] : -1;
        slot[tid] = s < a.num_slots ? s : -1;
    }
    float x[NC][8], sum = 0.f;
#pragma unroll
    for (int j = 0; j < NC; ++j) {
        const int c = 8 * (tid % 8) + 64 * j;
#pragma unroll
        for (int e = 0; e < 8; ++e) x[j][e] = 0.f;
        if (c < size) load_elems<8>(pr + c, x[j]);
#pragma unroll
        for (int e = 0; e < 8; ++e) sum += x[j][e] * x[j][e];
    }
#pragma unroll
    for (int m = 4; m >= 1; m >>= 1) sum += __shfl_xor(sum, m, 64);
    const float f = norm ? rsqrtf(sum / (float)size + a.eps) : 1.f;
#pragma unroll
    for (int j = 0; j < NC; ++j) {
#pragma unroll
        for (int e = 0; e < 8; ++e) x[j][e] *= f;
        store_elems<8>(tile + r * kRow + 8 * (tid % 8) + 64 * j, x[j]);
    }
    __syncthreads();
    // the tile of a slot, from the start of the pages, and the slot's place in it
    auto place = [&](int64_t s, int& token) {
        const int64_t block = s / a.block_size;
        const int off = (int)(s - block * a.block_size);
        token = off % kTileTokens;
        return ((block * a.kv_heads + h) * a.block_size + off - token) * pad;
    };
    if (is_key) {
        const int64_t s = slot[tid % 32];
        if (s < 0) return;
        int token;
        T* to = a.keys + place(s, token);
        for (int d = tid / 32 * 8; d < pad; d += 64) {
            float y[8];
            load_elems<8>(tile + tid % 32 * kRow + d, y);
            store_elems<8>(to + tile_key_entry(token, d), y);
        }
        return;
    }
    // runs of neighbouring tokens that do not leave a group of eight, taken in turn by 256 / pad sets of threads
    const int sets = 256 / pad, set = tid / pad, v = tid % pad;
    if (set >= sets) return;
    for (int first = 0, run = 0; first < 32; ++run) {
        const int64_t s = slot[first];
        int count = 1;
        while (first + count < 32 && (s + count) % 8 != 0 && slot[first + count] == s + count) ++count;
        if (s >= 0 && run % sets == set) {
            int token;
            T* to = a.values + place(s, token);
            to += tile_value_entry(token, v);
            if (count == 8) {
                float y[8];
#pragma unroll
                for (int e = 0; e < 8; ++e) y[e] = (float)tile[(first + e) * kRow + v];
                store_elems<8>(to, y);
            } else {
                for (int e = 0; e < count; ++e) to[e] = tile[(first + e) * kRow + v];
            }
        }
        first += count;
    }
}

template <class T, int LANES>
bool launch_vec(const HeadFrontArgs<T>& a, int64_t n, hipStream_t st) {
    const int per = 256 / LANES, nv = (num_vectors(a) + per - 1) / per;
    const dim3 grid((unsigned)n), block(256);
    if (nv <= 1) hipLaunchKernelGGL((head_front_kernel<T, LANES, 1>), grid, block, 0, st, a);
    else if (nv <= 2) hipLaunchKernelGGL((head_front_kernel<T, LANES, 2>), grid, block, 0, st, a);
    else if (nv <= 3) hipLaunchKernelGGL((head_front_kernel<T, LANES, 3>), grid, block, 0, st, a);
    else if (nv <= 6) hipLaunchKernelGGL((head_front_kernel<T, LANES, 6>), grid, block, 0, st, a);
    else return false;
    return true;
}

template <class T>
int launch(HeadFrontArgs<T> a, int64_t n, hipStream_t st) {
    const bool vec = a.dim % 8 == 0 && a.vdim % 8 == 0 && a.half % 8 == 0 && a.q_off % 8 == 0 && a.k_off % 8 == 0 && a.v_off % 8 == 0 &&
                     a.proj_stride % 8 == 0 && ptr_aligned(a.proj, 16) && ptr_aligned(a.keys, 16) && ptr_aligned(a.values, 16) && ptr_aligned(a.qx, 16) &&
                     ptr_aligned(a.bias, 16) && ptr_aligned(a.q_norm, 16) && ptr_aligned(a.k_norm, 16) && ptr_aligned(a.table, 16);
    bool done = false;
    // portions fill whole tiles; the rows of a decode batch belong to as many pages, and the main kernel writes them
    const bool portions = a.qx_rows < n ? n >= 64 : n >= 2048;
    if (vec && a.tiles && a.key_pad <= 256 && a.vdim_pad <= 256 && portions && a.kv_heads <= 32767) {
        const dim3 grid((unsigned)((n + 31) / 32), (unsigned)(2 * a.kv_heads)), block(256);
        const int pad = a.key_pad > a.vdim_pad ? a.key_pad : a.vdim_pad;
        if (pad <= 64) hipLaunchKernelGGL((fill_tiles_kernel<T, 1>), grid, block, 0, st, a, n);
        else if (pad <= 128) hipLaunchKernelGGL((fill_tiles_kernel<T, 2>), grid, block, 0, st, a, n);
        else hipLaunchKernelGGL((fill_tiles_kernel<T, 4>), grid, block, 0, st, a, n);
        a.apart = true;
    }
    const int longest = (a.norm_v || a.tiles) && !a.apart && a.vdim > a.dim ? a.vdim : a.dim;
    if (vec) {
        if (longest <= 32) done = launch_vec<T, 4>(a, n, st);
        else if (longest <= 64) done = launch_vec<T, 8>(a, n, st);
        else if (longest <= 128) done = launch_vec<T, 16>(a, n, st);
        else if (longest <= 256) done = launch_vec<T, 32>(a, n, st);
    }
    if (!done) hipLaunchKernelGGL((head_front_any_kernel<T>), dim3((unsigned)n), dim3(256), 0, st, a);
    return (int)hipGetLastError();
}

// the checks that both entries share, and the launch; `a` has everything but what is checked to fit an int
template <class T>
int run(const HeadFrontArgs<T>& a, int64_t n, void* stream) {
    if (n > 0x7fffffff) return INFER_KV_EINVAL;
    if (!a.proj || (!a.table && a.half) || !a.positions || !a.slots || !a.keys || !a.values || (a.qx_rows > 0 && !a.qx)) return INFER_KV_EINVAL;
    if (a.kv_heads > a.heads || a.maps * a.dim > a.key_pad || a.vdim > a.vdim_pad || 2 * a.half > a.dim || a.max_pos < 1 || a.num_slots < 0 ||
        a.qx_rows < 0 || a.qx_rows > n || (int64_t)a.heads * a.maps * a.key_pad > (1 << 24) || a.proj_stride > (1 << 24))
        return INFER_KV_EINVAL;
    if (a.q_off + (int64_t)a.heads * a.maps * a.dim > a.proj_stride || a.k_off + (int64_t)a.kv_heads * a.maps * a.dim > a.proj_stride ||
        a.v_off + (int64_t)a.kv_heads * a.vdim > a.proj_stride)
        return INFER_KV_EINVAL;
    return launch(a, n, (hipStream_t)stream);
}

bool sizes_valid(int64_t heads, int64_t kv_heads, int64_t maps, int64_t dim, int64_t vdim, int64_t q_off, int64_t k_off, int64_t v_off,
                 int64_t rot_dims, int64_t block_size, int64_t key_pad, int64_t vdim_pad) {
    return heads >= 1 && heads <= 4096 && kv_heads >= 1 && kv_heads <= 4096 && maps >= 1 && maps <= 2 && dim >= 1 && dim <= 65536 && vdim >= 1 &&
           vdim <= 65536 && key_pad >= 1 && key_pad <= 65536 && vdim_pad >= 1 && vdim_pad <= 65536 && rot_dims >= 0 && rot_dims % 2 == 0 &&
           rot_dims <= 65536 && block_size >= 1 && block_size <= (1 << 20) && q_off >= 0 && k_off >= 0 && v_off >= 0 && q_off <= (1 << 24) &&
           k_off <= (1 << 24) && v_off <= (1 << 24);
}

}  // namespace

extern "C" int infer_head_front(int elem, void* proj, int64_t proj_stride, int64_t heads, int64_t kv_heads, int64_t maps, int64_t dim,
                                int64_t vdim, int64_t q_off, int64_t k_off, int64_t v_off, const float* bias, const float* q_norm,
                                const float* k_norm, float eps, const float* table, int64_t rot_dims, int64_t max_pos,
                                const int64_t* positions, const int32_t* slots, void* cache, int64_t block_size, int64_t key_pad,
                                int64_t vdim_pad, int64_t num_slots, void* qx, int64_t qx_rows, int64_t n, void* stream) {
    if (n < 0 || !sizes_valid(heads, kv_heads, maps, dim, vdim, q_off, k_off, v_off, rot_dims, block_size, key_pad, vdim_pad) || !cache ||
        !q_norm != !k_norm)
        return INFER_KV_EINVAL;
    if (n == 0) return INFER_KV_OK;
    auto go = [&](auto zero) {
        using T = decltype(zero);
        const int row = (int)(key_pad + vdim_pad);
        const HeadFrontArgs<T> a{(T*)proj, proj_stride, (int)q_off, (int)k_off, (int)v_off, (int)heads, (int)kv_heads, (int)maps, (int)dim,
                                 (int)vdim, (int)(rot_dims / 2), bias, q_norm, k_norm, eps, q_norm != nullptr, false, 0.f, 0.0, table, max_pos,
                                 positions, slots, (T*)cache + vdim_pad, (T*)cache, row, row, false, false, (int)block_size, (int)key_pad, (int)vdim_pad,
                                 num_slots, (T*)qx, qx_rows};
        return run(a, n, stream);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}

extern "C" int infer_unit_head_front(int elem, void* proj, int64_t proj_stride, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim,
                                     int64_t q_off, int64_t k_off, int64_t v_off, float eps, int norm_values, float temp_coef,
                                     double temp_every, const int64_t* positions, const int32_t* slots, void* keys, void* values,
                                     int64_t block_size, int64_t key_pad, int64_t vdim_pad, int64_t num_slots, void* qx, int64_t qx_rows,
                                     int64_t n, void* stream) {
    if (n < 0 || !sizes_valid(heads, kv_heads, 1, dim, vdim, q_off, k_off, v_off, 0, block_size, key_pad, vdim_pad) || !(temp_every >= 0.0) || block_size % kTileTokens || key_pad % 32 || vdim_pad % 32)
        return INFER_KV_EINVAL;
    if (n == 0) return INFER_KV_OK;
    auto go = [&](auto zero) {
        using T = decltype(zero);
        const HeadFrontArgs<T> a{(T*)proj, proj_stride, (int)q_off, (int)k_off, (int)v_off, (int)heads, (int)kv_heads, 1, (int)dim, (int)vdim, 0,
                                 nullptr, nullptr, nullptr, eps, true, norm_values != 0, temp_coef, temp_every, nullptr, 1, positions, slots,
                                 (T*)keys, (T*)values, (int)key_pad, (int)vdim_pad, true, false, (int)block_size, (int)key_pad, (int)vdim_pad, num_slots,
                                 (T*)qx, qx_rows};
        return run(a, n, stream);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}
