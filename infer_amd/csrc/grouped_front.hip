// Front end of grouped attention over pages of [value | key] rows (row_attention.hip), for gfx950 (MI355X): per token
// the biases of the projections, an RMS norm over the whole q and the whole k projection, interleaved rotary positions
// on the first entries of every head, and the append of one cache row per key/value head.
//
// One workgroup per token; q and k are read once and stay in registers between the sum of squares and the rotation.
#include "elem.h"

namespace {

template <class T>
struct GroupedFrontArgs {
    T* proj; int64_t proj_stride;          // [q: heads x dim | ... k: kv_heads x dim at k_off | ... v: kv_heads x vdim at v_off | ...]
    int heads, kv_heads, dim, vdim, k_off, v_off, rot_pairs;    // kv_heads = 0: another layer has the keys
    const float* bias;                     // per column of proj, or nullptr
    const float* q_norm; const float* k_norm; float eps;        // nullptr: no norm
    const float* table; int64_t max_pos;   // [max_pos][rot_pairs][cos, sin]
    const int64_t* positions;
    const int32_t* slots;
    T* cache; int block_size, dim_pad, vdim_pad; int64_t num_slots;   // [blocks][kv_heads][block_size][vdim_pad + dim_pad]
    T* qx; int64_t qx_rows;                // rows below qx_rows: q to qx[row][head][dim_pad], others in place
};

// sums of two values over a workgroup of four wavefronts
__device__ __forceinline__ void block_sum2(float& x, float& y, float (*part)[4]) {
    x = wave_sum(x);
    y = wave_sum(y);
    if ((threadIdx.x & 63) == 0) {
        part[0][threadIdx.x >> 6] = x;
        part[1][threadIdx.x >> 6] = y;
    }
    __syncthreads();
    x = part[0][0] + part[0][1] + part[0][2] + part[0][3];
    y = part[1][0] + part[1][1] + part[1][2] + part[1][3];
}

template <class T, int N>
__device__ __forceinline__ void load_biased(const GroupedFrontArgs<T>& a, const T* pr, int col, float (&x)[N]) {
    load_elems<N>(pr + col, x);
    if (a.bias) {
        float b[N];
        load_elems<N>(a.bias + col, b);
#pragma unroll
        for (int e = 0; e < N; ++e) x[e] += b[e];
    }
}

template <class T>
__device__ __forceinline__ void rotate_pair(const GroupedFrontArgs<T>& a, const float* cs, int pair, float& u, float& v) {
    if (pair < a.rot_pairs) {
        const float c = cs[2 * pair], s = cs[2 * pair + 1], u0 = u;
        u = u0 * c - v * s;
        v = v * c + u0 * s;
    }
}

// the row of key/value head 0 in the cache, nullptr if the token has none; the next head's is block_size rows on
template <class T>
__device__ __forceinline__ T* cache_row(const GroupedFrontArgs<T>& a, int64_t slot) {
    if (a.kv_heads == 0 || slot < 0 || slot >= a.num_slots) return nullptr;
    const int64_t block = slot / a.block_size, off = slot - block * a.block_size;
    return a.cache + (block * a.kv_heads * a.block_size + off) * (a.dim_pad + a.vdim_pad);
}

// zeros behind the real sizes, which the attention kernels read
template <class T>
__device__ __forceinline__ void fill_padding(const GroupedFrontArgs<T>& a, T* row, int64_t head_rows, T* qx) {
    const int pad = a.dim_pad - a.dim, vpad = a.vdim_pad - a.vdim;
    if (row) {
        for (int i = threadIdx.x; i < a.kv_heads * pad; i += 256) row[i / pad * head_rows + a.vdim_pad + a.dim + i % pad] = (T)0.f;
        for (int i = threadIdx.x; i < a.kv_heads * vpad; i += 256) row[i / vpad * head_rows + a.vdim + i % vpad] = (T)0.f;
    }
    if (qx)
        for (int i = threadIdx.x; i < a.heads * pad; i += 256) qx[i / pad * a.dim_pad + a.dim + i % pad] = (T)0.f;
}

// NCH: chunks of eight columns of q, k and v per thread; everything is a multiple of eight.  SAME: 2048 columns, the
// distance between a thread's chunks, are whole heads, so that all its chunks of q and k start with the same pair.
template <class T, int NCH, bool SAME>
__global__ void __launch_bounds__(256) grouped_front_kernel(GroupedFrontArgs<T> a) {
    __shared__ float part[2][4];
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x;
    T* pr = a.proj + t * a.proj_stride;
    T* row = cache_row(a, a.slots[t]);
    int64_t pos = a.positions[t];
    pos = pos < 0 ? 0 : (pos >= a.max_pos ? a.max_pos - 1 : pos);
    const float* cs = a.table + pos * (2 * a.rot_pairs);
    const int64_t head_rows = (int64_t)a.block_size * (a.dim_pad + a.vdim_pad);
    const int nq = a.heads * a.dim / 8, nk = row ? a.kv_heads * a.dim / 8 : 0, total = nq + nk + (row ? a.kv_heads * a.vdim / 8 : 0);
    // cosine and sine of four pairs from p on
    auto turn_of = [&](int p, float (&turn)[8]) {
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            turn[2 * k] = 1.f;
            turn[2 * k + 1] = 0.f;
            if (p + k < a.rot_pairs) {
                const float2 v = *reinterpret_cast<const float2*>(cs + 2 * (p + k));
                turn[2 * k] = v.x;
                turn[2 * k + 1] = v.y;
            }
        }
    };
    float x[NCH][8], turn[8], sq = 0.f, sk = 0.f;
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
        const int i = tid + 256 * j;
        if (i < total) load_biased(a, pr, i < nq ? 8 * i : i < nq + nk ? a.k_off + 8 * (i - nq) : a.v_off + 8 * (i - nq - nk), x[j]);
    }
    if constexpr (SAME) turn_of(8 * tid % a.dim / 2, turn);
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
        const int i = tid + 256 * j;
        float s = 0.f;
        if (i < nq + nk)
#pragma unroll
            for (int e = 0; e < 8; ++e) s += x[j][e] * x[j][e];
        sq += i < nq ? s : 0.f;
        sk += i < nq ? 0.f : s;
    }
    block_sum2(sq, sk, part);
    const float rq = rsqrtf(sq / (float)(8 * nq) + a.eps), rk = rsqrtf(sk / (float)(8 * (nk > 0 ? nk : 1)) + a.eps);
    T* qx = t < a.qx_rows ? a.qx + t * a.heads * a.dim_pad : nullptr;
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
        const int i = tid + 256 * j;
        if (i >= total) continue;
        T* to;
        if (i < nq + nk) {
            const bool is_q = i < nq;
            const int col = 8 * (is_q ? i : i - nq);
            const float* norm = is_q ? a.q_norm : a.k_norm;
            if (norm) {
                float w[8];
                load_elems<8>(norm + col, w);
#pragma unroll
                for (int e = 0; e < 8; ++e) x[j][e] *= (is_q ? rq : rk) * w[e];
            }
            if constexpr (!SAME) turn_of(col % a.dim / 2, turn);
#pragma unroll
            for (int e = 0; e < 8; e += 2) {
                const float u = x[j][e], v = x[j][e + 1];
                x[j][e] = u * turn[e] - v * turn[e + 1];
                x[j][e + 1] = v * turn[e] + u * turn[e + 1];
            }
            if (is_q && !qx) {
                to = pr + col;
            } else {
                const int h = col / a.dim, d = col - h * a.dim;
                to = is_q ? qx + h * a.dim_pad + d : row + h * head_rows + a.vdim_pad + d;
            }
        } else {
            const int col = 8 * (i - nq - nk), h = col / a.vdim;
            to = row + h * head_rows + (col - h * a.vdim);
        }
        store_elems<8>(to, x[j]);
    }
    fill_padding(a, row, head_rows, qx);
}

// any size: one pair of entries at a time (the last one alone if dim is odd), everything read twice
template <class T>
__global__ void __launch_bounds__(256) grouped_front_any_kernel(GroupedFrontArgs<T> a) {
    __shared__ float part[2][4];
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x;
    T* pr = a.proj + t * a.proj_stride;
    int64_t pos = a.positions[t];
    pos = pos < 0 ? 0 : (pos >= a.max_pos ? a.max_pos - 1 : pos);
    const float* cs = a.table + pos * (2 * a.rot_pairs);
    T* row = cache_row(a, a.slots[t]);
    const int64_t head_rows = (int64_t)a.block_size * (a.dim_pad + a.vdim_pad);
    const int nq = a.heads * a.dim, nk = row ? a.kv_heads * a.dim : 0;
    float sq = 0.f, sk = 0.f;
    for (int i = tid; i < nq + nk; i += 256) {
        float x[1];
        load_biased(a, pr, i < nq ? i : a.k_off + i - nq, x);
        (i < nq ? sq : sk) += x[0] * x[0];
    }
    block_sum2(sq, sk, part);
    const float rq = rsqrtf(sq / (float)nq + a.eps), rk = rsqrtf(sk / (float)(nk > 0 ? nk : 1) + a.eps);
    T* qx = t < a.qx_rows ? a.qx + t * a.heads * a.dim_pad : nullptr;
    const int pairs = (a.dim + 1) / 2, hk = row ? a.kv_heads : 0;
    for (int i = tid; i < (a.heads + hk) * pairs; i += 256) {
        const bool is_q = i < a.heads * pairs;
        const int h = is_q ? i / pairs : i / pairs - a.heads, p = i % pairs, col = h * a.dim + 2 * p;
        const bool both = 2 * p + 1 < a.dim;
        const float* norm = is_q ? a.q_norm : a.k_norm;
        const int from = (is_q ? 0 : a.k_off) + col;
        float x[1], y[1] = {0.f};
        load_biased(a, pr, from, x);
        if (both) load_biased(a, pr, from + 1, y);
        if (norm) {
            x[0] *= (is_q ? rq : rk) * norm[col];
            if (both) y[0] *= (is_q ? rq : rk) * norm[col + 1];
        }
        rotate_pair(a, cs, p, x[0], y[0]);
        T* to = !is_q ? row + h * head_rows + a.vdim_pad + 2 * p : qx ? qx + h * a.dim_pad + 2 * p : pr + col;
        to[0] = (T)x[0];
        if (both) to[1] = (T)y[0];
    }
    if (row)
        for (int i = tid; i < a.kv_heads * a.vdim; i += 256) {
            float v[1];
            load_biased(a, pr, a.v_off + i, v);
            row[i / a.vdim * head_rows + i % a.vdim] = (T)v[0];
        }
    fill_padding(a, row, head_rows, qx);
}

template <class T>
int launch(const GroupedFrontArgs<T>& a, int64_t n, hipStream_t st) {
    const bool vec = a.dim % 8 == 0 && a.vdim % 8 == 0 && a.k_off % 8 == 0 && a.v_off % 8 == 0 && a.proj_stride % 8 == 0 &&
                     ptr_aligned(a.proj, 16) && ptr_aligned(a.cache, 16) && ptr_aligned(a.qx, 16) && ptr_aligned(a.bias, 16) &&
                     ptr_aligned(a.q_norm, 16) && ptr_aligned(a.k_norm, 16) && ptr_aligned(a.table, 8);
    const int chunks = ((a.heads + a.kv_heads) * a.dim / 8 + a.kv_heads * a.vdim / 8 + 255) / 256;
    const dim3 grid((unsigned)n), block(256);
#define GO(N) \
    do { \
        if (2048 % a.dim == 0) hipLaunchKernelGGL((grouped_front_kernel<T, N, true>), grid, block, 0, st, a); \
        else hipLaunchKernelGGL((grouped_front_kernel<T, N, false>), grid, block, 0, st, a); \
    } while (0)
    if (vec && chunks <= 1) GO(1);
    else if (vec && chunks <= 2) GO(2);
    else if (vec && chunks <= 3) GO(3);
    else if (vec && chunks <= 6) GO(6);
    else hipLaunchKernelGGL((grouped_front_any_kernel<T>), grid, block, 0, st, a);
#undef GO
    return (int)hipGetLastError();
}

}  // namespace

extern "C" int infer_grouped_front(int elem, void* proj, int64_t proj_stride, int64_t heads, int64_t kv_heads, int64_t dim,
                                   int64_t vdim, int64_t k_off, int64_t v_off, const float* bias, const float* q_norm,
                                   const float* k_norm, float eps, const float* table, int64_t rot_dims, int64_t max_pos,
                                   const int64_t* positions, const int32_t* slots, void* cache, int64_t block_size,
                                   int64_t dim_pad, int64_t vdim_pad, int64_t num_slots, void* qx, int64_t qx_rows, int64_t n,
                                   void* stream) {
    if (n < 0 || n > 0x7fffffff) return INFER_KV_EINVAL;
    if (n == 0) return INFER_KV_OK;
    if (!proj || (!table && rot_dims) || !positions || !slots || (kv_heads > 0 && !cache) || (qx_rows > 0 && !qx)) return INFER_KV_EINVAL;
    if (heads < 1 || heads > 4096 || kv_heads < 0 || kv_heads > heads || dim < 1 || dim > dim_pad || dim_pad > 65536 || vdim < 1 ||
        vdim > vdim_pad || vdim_pad > 65536 || rot_dims < 0 || rot_dims % 2 || rot_dims > dim || max_pos < 1 || block_size < 1 ||
        block_size > (1 << 20) || num_slots < 0 || qx_rows < 0 || qx_rows > n || heads * dim > (1 << 24))
        return INFER_KV_EINVAL;
    if (proj_stride < heads * dim || (kv_heads > 0 && (k_off < heads * dim || v_off < k_off + kv_heads * dim || proj_stride < v_off + kv_heads * vdim)))
        return INFER_KV_EINVAL;
    if (kv_heads == 0) k_off = v_off = 0;
    auto go = [&](auto zero) {
        using T = decltype(zero);
        const GroupedFrontArgs<T> a{(T*)proj, proj_stride, (int)heads, (int)kv_heads, (int)dim, (int)vdim, (int)k_off, (int)v_off,
                                    (int)(rot_dims / 2), bias, q_norm, k_norm, eps, table, max_pos, positions, slots, (T*)cache,
                                    (int)block_size, (int)dim_pad, (int)vdim_pad, num_slots, (T*)qx, qx_rows};
        return launch(a, n, (hipStream_t)stream);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}
