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
//
// The attention itself is in row_attention.hip (query rows against cached rows) and dense_prefill.hip.
#include "elem.h"

namespace {

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

