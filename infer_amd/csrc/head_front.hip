// Front end of masked attention over pages of [value | key] rows (row_attention.hip), for gfx950 (MI355X): per token
// the biases of the projections, an RMS norm over every head's query and key, rotary positions (entry i turns with
// entry i + half), and the append of one cache row per key/value head.
//
// A head may have two maps: two queries and two keys beside one value.  Each map is a vector of its own here.  The cached
// row is [value | key of map 1 | key of map 2], and a query that goes to the row kernels is padded to the length of both keys,
// with zeros where the other map's key stands.
#include "elem.h"

namespace {

template <class T>
struct HeadFrontArgs {
    T* proj; int64_t proj_stride; int q_off, k_off, v_off;   // heads x maps x dim, kv_heads x maps x dim, kv_heads x vdim
    int heads, kv_heads, maps, dim, vdim, half;              // half: rotated pairs
    const float* bias;                     // per column of proj, or nullptr
    const float* q_norm; const float* k_norm; float eps;     // [dim], nullptr: no norm
    const float* table; int64_t max_pos;   // [max_pos][half][cos, sin]
    const int64_t* positions;
    const int32_t* slots;
    T* cache; int block_size, key_pad, vdim_pad; int64_t num_slots;   // [blocks][kv_heads][block_size][vdim_pad + key_pad]
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

// the row of key/value head 0 in the cache, nullptr if the token has none; the next head's is block_size rows on
template <class T>
__device__ __forceinline__ T* cache_row(const HeadFrontArgs<T>& a, int64_t slot) {
    if (slot < 0 || slot >= a.num_slots) return nullptr;
    const int64_t block = slot / a.block_size, off = slot - block * a.block_size;
    return a.cache + (block * a.kv_heads * a.block_size + off) * (a.key_pad + a.vdim_pad);
}

// where vector i (queries first, then keys) of a token comes from and goes to; to == nullptr: nowhere
template <class T>
struct Place { int from; T* to; const float* norm; };
template <class T>
__device__ __forceinline__ Place<T> place_of(const HeadFrontArgs<T>& a, T* pr, T* row, int64_t head_rows, T* qx, int i) {
    const int nq = a.heads * a.maps;
    if (i < nq) {
        const int from = a.q_off + i * a.dim;
        return {from, qx ? qx + (int64_t)i * a.key_pad + i % a.maps * a.dim : pr + from, a.q_norm};
    }
    i -= nq;
    return {a.k_off + i * a.dim, row ? row + i / a.maps * head_rows + a.vdim_pad + i % a.maps * a.dim : nullptr, a.k_norm};
}

// zeros that the attention kernels read: behind the real sizes, and at the other map's place in a query
template <class T>
__device__ __forceinline__ void fill_padding(const HeadFrontArgs<T>& a, T* row, int64_t head_rows, T* qx) {
    const int used = a.maps * a.dim, pad = a.key_pad - used, vpad = a.vdim_pad - a.vdim;
    if (row) {
        for (int i = threadIdx.x; i < a.kv_heads * pad; i += 256) row[i / pad * head_rows + a.vdim_pad + used + i % pad] = (T)0.f;
        for (int i = threadIdx.x; i < a.kv_heads * vpad; i += 256) row[i / vpad * head_rows + a.vdim + i % vpad] = (T)0.f;
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
    T* row = cache_row(a, a.slots[t]);
    T* qx = t < a.qx_rows ? a.qx + t * a.heads * a.maps * a.key_pad : nullptr;
    const int64_t head_rows = (int64_t)a.block_size * (a.key_pad + a.vdim_pad);
    const int total = (a.heads + a.kv_heads) * a.maps;
    int64_t pos = a.positions[t];
    pos = pos < 0 ? 0 : (pos >= a.max_pos ? a.max_pos - 1 : pos);
    const bool in = c < a.dim, low = c < a.half, turned = c < 2 * a.half;
    float x[NV][8];
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int i = tid / LANES + j * (256 / LANES);
#pragma unroll
        for (int e = 0; e < 8; ++e) x[j][e] = 0.f;
        if (in && i < total) load_biased(a, pr, place_of(a, pr, row, head_rows, qx, i).from + c, x[j]);
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
    // values
    if (row)
        for (int i = tid; i < a.kv_heads * a.vdim / 8; i += 256) {
            float v[8];
            load_biased(a, pr, a.v_off + 8 * i, v);
            const int h = 8 * i / a.vdim;
            store_elems<8>(row + h * head_rows + (8 * i - h * a.vdim), v);
        }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int i = tid / LANES + j * (256 / LANES);
        const Place<T> p = place_of(a, pr, row, head_rows, qx, i < total ? i : 0);
        if (p.norm) {
            float s = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) s += x[j][e] * x[j][e];
#pragma unroll
            for (int m = LANES / 2; m >= 1; m >>= 1) s += __shfl_xor(s, m, 64);
            const float r = rsqrtf(s / (float)a.dim + a.eps);
            if (in) {
                float w[8];
                load_elems<8>(p.norm + c, w);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[j][e] *= r * w[e];
            }
        }
        if (a.half > 0) {
            const int other = (tid & 63) + (low ? a.half / 8 : turned ? -(a.half / 8) : 0);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float y = __shfl(x[j][e], other, 64);
                if (turned) x[j][e] = x[j][e] * turn[2 * e] + (low ? -y : y) * turn[2 * e + 1];
            }
        }
        if (in && i < total && p.to) store_elems<8>(p.to + c, x[j]);
    }
    fill_padding(a, row, head_rows, qx);
}

// any size: one wavefront per vector
template <class T>
__global__ void __launch_bounds__(256) head_front_any_kernel(HeadFrontArgs<T> a) {
    const int64_t t = blockIdx.x;
    const int lane = threadIdx.x & 63;
    T* pr = a.proj + t * a.proj_stride;
    T* row = cache_row(a, a.slots[t]);
    T* qx = t < a.qx_rows ? a.qx + t * a.heads * a.maps * a.key_pad : nullptr;
    const int64_t head_rows = (int64_t)a.block_size * (a.key_pad + a.vdim_pad);
    int64_t pos = a.positions[t];
    pos = pos < 0 ? 0 : (pos >= a.max_pos ? a.max_pos - 1 : pos);
    const float* cs = a.table + pos * (2 * a.half);
    for (int i = threadIdx.x >> 6; i < (a.heads + a.kv_heads) * a.maps; i += 4) {
        const Place<T> p = place_of(a, pr, row, head_rows, qx, i);
        float r = 1.f;
        if (p.norm) {
            float s = 0.f, x[1];
            for (int d = lane; d < a.dim; d += 64) {
                load_biased(a, pr, p.from + d, x);
                s += x[0] * x[0];
            }
            r = rsqrtf(wave_sum(s) / (float)a.dim + a.eps);
        }
        if (!p.to) continue;
        // a pair is read and written by one lane
        for (int d = lane; d < a.dim - a.half; d += 64) {
            const bool pair = d < a.half;
            const int at = pair ? d : d + a.half;
            float u[1], v[1] = {0.f};
            load_biased(a, pr, p.from + at, u);
            if (p.norm) u[0] *= r * p.norm[at];
            if (pair) {
                load_biased(a, pr, p.from + d + a.half, v);
                if (p.norm) v[0] *= r * p.norm[d + a.half];
                const float co = cs[2 * d], si = cs[2 * d + 1];
                p.to[d + a.half] = (T)(v[0] * co + u[0] * si);
                u[0] = u[0] * co - v[0] * si;
            }
            p.to[at] = (T)u[0];
        }
    }
    if (row)
        for (int i = threadIdx.x; i < a.kv_heads * a.vdim; i += 256) {
            float v[1];
            load_biased(a, pr, a.v_off + i, v);
            row[i / a.vdim * head_rows + i % a.vdim] = (T)v[0];
        }
    fill_padding(a, row, head_rows, qx);
}

template <class T, int LANES>
bool launch_vec(const HeadFrontArgs<T>& a, int64_t n, hipStream_t st) {
    const int per = 256 / LANES, nv = ((a.heads + a.kv_heads) * a.maps + per - 1) / per;
    const dim3 grid((unsigned)n), block(256);
    if (nv <= 1) hipLaunchKernelGGL((head_front_kernel<T, LANES, 1>), grid, block, 0, st, a);
    else if (nv <= 2) hipLaunchKernelGGL((head_front_kernel<T, LANES, 2>), grid, block, 0, st, a);
    else if (nv <= 3) hipLaunchKernelGGL((head_front_kernel<T, LANES, 3>), grid, block, 0, st, a);
    else if (nv <= 6) hipLaunchKernelGGL((head_front_kernel<T, LANES, 6>), grid, block, 0, st, a);
    else return false;
    return true;
}

template <class T>
int launch(const HeadFrontArgs<T>& a, int64_t n, hipStream_t st) {
    const bool vec = a.dim % 8 == 0 && a.vdim % 8 == 0 && a.half % 8 == 0 && a.q_off % 8 == 0 && a.k_off % 8 == 0 && a.v_off % 8 == 0 &&
                     a.proj_stride % 8 == 0 && ptr_aligned(a.proj, 16) && ptr_aligned(a.cache, 16) && ptr_aligned(a.qx, 16) &&
                     ptr_aligned(a.bias, 16) && ptr_aligned(a.q_norm, 16) && ptr_aligned(a.k_norm, 16) && ptr_aligned(a.table, 16);
    bool done = false;
    if (vec) {
        if (a.dim <= 32) done = launch_vec<T, 4>(a, n, st);
        else if (a.dim <= 64) done = launch_vec<T, 8>(a, n, st);
        else if (a.dim <= 128) done = launch_vec<T, 16>(a, n, st);
        else if (a.dim <= 256) done = launch_vec<T, 32>(a, n, st);
    }
    if (!done) hipLaunchKernelGGL((head_front_any_kernel<T>), dim3((unsigned)n), dim3(256), 0, st, a);
    return (int)hipGetLastError();
}

}  // namespace

extern "C" int infer_head_front(int elem, void* proj, int64_t proj_stride, int64_t heads, int64_t kv_heads, int64_t maps, int64_t dim,
                                int64_t vdim, int64_t q_off, int64_t k_off, int64_t v_off, const float* bias, const float* q_norm,
                                const float* k_norm, float eps, const float* table, int64_t rot_dims, int64_t max_pos,
                                const int64_t* positions, const int32_t* slots, void* cache, int64_t block_size, int64_t key_pad,
                                int64_t vdim_pad, int64_t num_slots, void* qx, int64_t qx_rows, int64_t n, void* stream) {
    if (n < 0 || n > 0x7fffffff) return INFER_KV_EINVAL;
    if (n == 0) return INFER_KV_OK;
    if (!proj || (!table && rot_dims) || !positions || !slots || !cache || (qx_rows > 0 && !qx)) return INFER_KV_EINVAL;
    if (heads < 1 || heads > 4096 || kv_heads < 1 || kv_heads > heads || maps < 1 || maps > 2 || dim < 1 || dim > 65536 ||
        maps * dim > key_pad || key_pad > 65536 || vdim < 1 || vdim > vdim_pad || vdim_pad > 65536 || rot_dims < 0 || rot_dims % 2 ||
        rot_dims > dim || max_pos < 1 || block_size < 1 || block_size > (1 << 20) || num_slots < 0 || qx_rows < 0 || qx_rows > n ||
        heads * maps * key_pad > (1 << 24) || proj_stride > (1 << 24))
        return INFER_KV_EINVAL;
    if (q_off < 0 || k_off < 0 || v_off < 0 || q_off + heads * maps * dim > proj_stride || k_off + kv_heads * maps * dim > proj_stride ||
        v_off + kv_heads * vdim > proj_stride)
        return INFER_KV_EINVAL;
    auto go = [&](auto zero) {
        using T = decltype(zero);
        const HeadFrontArgs<T> a{(T*)proj, proj_stride, (int)q_off, (int)k_off, (int)v_off, (int)heads, (int)kv_heads, (int)maps, (int)dim,
                                 (int)vdim, (int)(rot_dims / 2), bias, q_norm, k_norm, eps, table, max_pos, positions, slots, (T*)cache,
                                 (int)block_size, (int)key_pad, (int)vdim_pad, num_slots, (T*)qx, qx_rows};
        return launch(a, n, (hipStream_t)stream);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}
