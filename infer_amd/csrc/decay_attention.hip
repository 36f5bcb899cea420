// Linear attention with a constant decay per head, for gfx950 (MI355X).  Per head, over a float32 state S[dim][vdim]:
//     S <- d S + k v^T ;   o = c S^T q
// (d and c constants), q, k and v being projections, optionally behind silu (q, k, v) or a rotary embedding (q, k;
// entry i turns with entry i + pairs).  Behind it an RMS norm over each head or over all heads at once and an output gate.
//
//   decay_step_kernel     one token per sequence (decode): one workgroup per (sequence, head), the state passes
//                         through registers once; with a norm per head the norm and the gate are in it too
//   decay_scan_any_kernel prompt portions of any size and element type, token by token
//   decay_out_kernel      norm and gate of whole rows
//
// A sequence at position 0 starts from a zero state whatever its slot holds, so a slot needs no clearing when another
// sequence takes it over.  d is held as a sum of two floats: its rounding error would enter a long memory once per
// token.
#include "elem.h"

namespace {

constexpr int kThreads = 256;

template <class T>
struct DecayArgs {
    const T* proj; int64_t proj_stride; int q_off, k_off, v_off;      // heads x dim, heads x dim, heads x vdim
    int heads, dim, vdim, dim_pad, vdim_pad;
    const float* decay;                    // [3][heads]: d rounded to float, what is missing, log2 d
    bool silu;
    const float* table; int rot_pairs; int64_t max_pos;               // [max_pos][rot_pairs][cos, sin]
    float scale;                           // c
    float* state; int num_slots;           // [slots][heads][dim_pad][vdim_pad]
    T* o; int64_t o_stride;                // [row][heads * vdim]
};

template <class T>
struct DecayOutArgs {
    const T* o; int64_t o_stride;          // [row][heads * vdim]
    const T* gate; int64_t gate_stride;    // the same columns
    const float* norm;                     // [heads * vdim] or nullptr
    bool gate_silu;                        // silu or sigmoid
    int heads, vdim;
    float eps;
    T* out; int64_t out_stride;
};

template <class T>
__device__ __forceinline__ float gate_of(const DecayOutArgs<T>& a, float z) { return a.gate_silu ? silu_f(z) : sigmoid_f(z); }

template <class T>
__device__ __forceinline__ const float* table_row(const DecayArgs<T>& a, int64_t pos) {
    pos = pos < 0 ? 0 : (pos >= a.max_pos ? a.max_pos - 1 : pos);
    return a.table + pos * (2 * a.rot_pairs);
}

// entry d of the projection that starts at p, behind silu or rotation
template <class T>
__device__ __forceinline__ float entry(const DecayArgs<T>& a, const T* p, const float* cs, int d) {
    const float x = (float)p[d];
    if (a.silu) return silu_f(x);
    if (d >= 2 * a.rot_pairs) return x;
    const bool low = d < a.rot_pairs;
    const int i = low ? d : d - a.rot_pairs;
    const float y = (float)p[low ? d + a.rot_pairs : i];
    return low ? x * cs[2 * i] - y * cs[2 * i + 1] : x * cs[2 * i] + y * cs[2 * i + 1];
}

// ------------------------------------------------------------------ any size
struct Span { int32_t row0, count, slot, pos0; };       // consecutive tokens of one sequence

// One workgroup per (16 columns of the state, head, span); thread (r, c): column c, state rows r, r + 16, ...
template <class T>
__global__ void __launch_bounds__(kThreads) decay_scan_any_kernel(DecayArgs<T> a, const Span* spans, const int32_t* slots,
                                                                  const int64_t* positions) {
    extern __shared__ float sh[];
    float* s = sh;                              // [dim_pad][16]
    float* qs = s + a.dim_pad * 16;             // [dim_pad]
    float* ks = qs + a.dim_pad;
    float* part = ks + a.dim_pad;               // [4][16]
    const int tid = threadIdx.x, c = tid & 15, r = tid >> 4, h = blockIdx.y, v = blockIdx.x * 16 + c;
    const Span p = spans ? spans[blockIdx.z] : Span{(int32_t)blockIdx.z, 1, slots[blockIdx.z], (int32_t)positions[blockIdx.z]};
    if (p.slot < 0 || p.slot >= a.num_slots) {           // a padding row of a captured batch
        if (r == 0 && v < a.vdim)
            for (int t = 0; t < p.count; ++t) a.o[(int64_t)(p.row0 + t) * a.o_stride + (int64_t)h * a.vdim + v] = (T)0.f;
        return;
    }
    float* sp = a.state + (((int64_t)p.slot * a.heads + h) * a.dim_pad) * a.vdim_pad + v;
    for (int d = r; d < a.dim_pad; d += 16) s[d * 16 + c] = p.pos0 > 0 ? sp[(int64_t)d * a.vdim_pad] : 0.f;
    const float hi = a.decay[h], lo = a.decay[a.heads + h];
    for (int t = 0; t < p.count; ++t) {
        const T* row = a.proj + (int64_t)(p.row0 + t) * a.proj_stride;
        const float* cs = table_row(a, p.pos0 + t);
        for (int d = tid; d < a.dim_pad; d += kThreads) {
            qs[d] = d < a.dim ? entry(a, row + a.q_off + h * a.dim, cs, d) : 0.f;
            ks[d] = d < a.dim ? entry(a, row + a.k_off + h * a.dim, cs, d) : 0.f;
        }
        float x = v < a.vdim ? (float)row[a.v_off + h * a.vdim + v] : 0.f;
        if (a.silu) x = silu_f(x);
        __syncthreads();
        float o = 0.f;
        for (int d = r; d < a.dim_pad; d += 16) {
            const float y = s[d * 16 + c];
            const float z = fmaf(y, hi, fmaf(y, lo, ks[d] * x));
            s[d * 16 + c] = z;
            o += z * qs[d];
        }
        o += __shfl_xor(o, 16, 64);
        o += __shfl_xor(o, 32, 64);
        if ((tid & 63) < 16) part[(tid >> 6) * 16 + c] = o;
        __syncthreads();
        if (tid < 16 && v < a.vdim)
            a.o[(int64_t)(p.row0 + t) * a.o_stride + (int64_t)h * a.vdim + v] =
                (T)((part[c] + part[16 + c] + part[32 + c] + part[48 + c]) * a.scale);
    }
    for (int d = r; d < a.dim_pad; d += 16) sp[(int64_t)d * a.vdim_pad] = s[d * 16 + c];
}

// ------------------------------------------------------------------ one token per sequence
// Thread (r, c): column group c (four columns of the state), rows r, r + R, ...; NP rows per thread.
template <class T, int NP, bool FUSED>
__global__ void __launch_bounds__(kThreads) decay_step_kernel(DecayArgs<T> a, DecayOutArgs<T> b, const int32_t* slots, const int64_t* positions) {
    extern __shared__ __attribute__((aligned(16))) float sh[];
    const int row = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    const int slot = slots[row];
    T* out = (FUSED ? b.out + (int64_t)row * b.out_stride : a.o + (int64_t)row * a.o_stride) + (int64_t)h * a.vdim;
    if (slot < 0 || slot >= a.num_slots) {
        for (int v = tid; v < a.vdim; v += kThreads) out[v] = (T)0.f;
        return;
    }
    const int64_t pos = positions[row];
    const int cgs = a.vdim_pad / 4, rgs = kThreads / cgs;
    float* ks = sh;                                  // [dim_pad]
    float* qs = ks + a.dim_pad;
    float* vs = qs + a.dim_pad;                      // [vdim_pad]
    float* red = vs + a.vdim_pad;                    // [rgs][vdim_pad]
    float* part = red + rgs * a.vdim_pad;            // [4]
    const int cg = tid % cgs, rg = tid / cgs;
    const bool works = rg < rgs;
    float* sp = a.state + (((int64_t)slot * a.heads + h) * a.dim_pad) * a.vdim_pad + 4 * cg;
    f32x4_t s[NP];
    if (works)
#pragma unroll
        for (int i = 0; i < NP; ++i) {
            const int d = rg + i * rgs;
            s[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
            if (pos > 0 && d < a.dim_pad) s[i] = *reinterpret_cast<const f32x4_t*>(sp + (int64_t)d * a.vdim_pad);
        }
    const T* in = a.proj + (int64_t)row * a.proj_stride;
    const float* cs = table_row(a, pos);
    for (int d = tid; d < a.dim_pad; d += kThreads) {
        qs[d] = d < a.dim ? entry(a, in + a.q_off + h * a.dim, cs, d) : 0.f;
        ks[d] = d < a.dim ? entry(a, in + a.k_off + h * a.dim, cs, d) : 0.f;
    }
    for (int v = tid; v < a.vdim_pad; v += kThreads) {
        float x = v < a.vdim ? (float)in[a.v_off + h * a.vdim + v] : 0.f;
        vs[v] = a.silu ? silu_f(x) : x;
    }
    const float hi = a.decay[h], lo = a.decay[a.heads + h];
    __syncthreads();
    if (works) {
        const f32x4_t x = *reinterpret_cast<const f32x4_t*>(vs + 4 * cg);
        f32x4_t o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < NP; ++i) {
            const int d = rg + i * rgs;
            if (d < a.dim_pad) {
                const float k = ks[d], q = qs[d];
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    s[i][e] = fmaf(s[i][e], hi, fmaf(s[i][e], lo, k * x[e]));
                    o[e] = fmaf(s[i][e], q, o[e]);
                }
                *reinterpret_cast<f32x4_t*>(sp + (int64_t)d * a.vdim_pad) = s[i];
            }
        }
        *reinterpret_cast<f32x4_t*>(red + rg * a.vdim_pad + 4 * cg) = o * a.scale;
    }
    __syncthreads();
    f32x4_t y = {0.f, 0.f, 0.f, 0.f};
    if (tid < cgs)
        for (int r = 0; r < rgs; ++r) y += *reinterpret_cast<const f32x4_t*>(red + r * a.vdim_pad + 4 * tid);
    if constexpr (FUSED) {
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < 4; ++e) ss += y[e] * y[e];           // padded columns are zero
        const float rs = rsqrtf(block_sum<4>(ss, part) / (float)a.vdim + b.eps);
        if (tid < cgs) {
            const T* g = b.gate + (int64_t)row * b.gate_stride + (int64_t)h * a.vdim;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int v = 4 * tid + e;
                if (v < a.vdim) y[e] *= rs * (b.norm ? b.norm[h * a.vdim + v] : 1.f) * gate_of(b, (float)g[v]);
            }
        }
    }
    if (tid < cgs)
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (4 * tid + e < a.vdim) out[4 * tid + e] = (T)y[e];
}

// ------------------------------------------------------------------ norm and gate
// One norm over the whole row.  NCH: chunks of VEC columns per thread, kept in registers.
template <class T, int VEC, int NCH>
__global__ void __launch_bounds__(kThreads) decay_out_row_kernel(DecayOutArgs<T> a) {
    __shared__ float part[4];
    const int64_t row = blockIdx.x;
    const int n = a.heads * a.vdim;
    float x[NCH][VEC], ss = 0.f;
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
        const int c = (threadIdx.x + j * kThreads) * VEC;
        if (c < n) {
            load_elems<VEC>(a.o + row * a.o_stride + c, x[j]);
#pragma unroll
            for (int e = 0; e < VEC; ++e) ss += x[j][e] * x[j][e];
        }
    }
    const float rs = rsqrtf(block_sum<4>(ss, part) / (float)n + a.eps);
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
        const int c = (threadIdx.x + j * kThreads) * VEC;
        if (c < n) {
            float g[VEC], w[VEC];
            load_elems<VEC>(a.gate + row * a.gate_stride + c, g);
            if (a.norm) load_elems<VEC>(a.norm + c, w);
#pragma unroll
            for (int e = 0; e < VEC; ++e) x[j][e] *= rs * (a.norm ? w[e] : 1.f) * gate_of(a, g[e]);
            store_elems<VEC>(a.out + row * a.out_stride + c, x[j]);
        }
    }
}

// A norm per head.  LANES lanes share a head, four values each (vdim = 4 LANES); LANES = 0: any vdim, one wavefront per head.
template <class T, int LANES>
__global__ void __launch_bounds__(kThreads) decay_out_heads_kernel(DecayOutArgs<T> a) {
    const int64_t row = blockIdx.x;
    const T* o = a.o + row * a.o_stride;
    const T* gate = a.gate + row * a.gate_stride;
    T* out = a.out + row * a.out_stride;
    if constexpr (LANES > 0) {
        const int n = a.heads * a.vdim;
        for (int c = 4 * threadIdx.x; c < n; c += 4 * kThreads) {        // a head's lanes are in the loop together: n is a multiple of 4 LANES
            float x[4], g[4], w[4];
            load_elems<4>(o + c, x);
            load_elems<4>(gate + c, g);
            if (a.norm) load_elems<4>(a.norm + c, w);
            float ss = x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
#pragma unroll
            for (int m = LANES / 2; m >= 1; m >>= 1) ss += __shfl_xor(ss, m, 64);
            const float rs = rsqrtf(ss / (float)a.vdim + a.eps);
#pragma unroll
            for (int e = 0; e < 4; ++e) x[e] *= rs * (a.norm ? w[e] : 1.f) * gate_of(a, g[e]);
            store_elems<4>(out + c, x);
        }
    } else {
        const int lane = threadIdx.x & 63;
        for (int h = threadIdx.x >> 6; h < a.heads; h += 4) {
            float ss = 0.f;
            for (int v = lane; v < a.vdim; v += 64) {
                const float x = (float)o[h * a.vdim + v];
                ss += x * x;
            }
            const float rs = rsqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
            for (int v = lane; v < a.vdim; v += 64) {
                const int c = h * a.vdim + v;
                out[c] = (T)((float)o[c] * rs * (a.norm ? a.norm[c] : 1.f) * gate_of(a, (float)gate[c]));
            }
        }
    }
}

template <class T>
int launch_out(const DecayOutArgs<T>& a, bool per_head, int64_t rows, hipStream_t st) {
    const size_t four = 4 * sizeof(T);
    const int n = a.heads * a.vdim;
    const bool vec = a.vdim % 4 == 0 && a.o_stride % 4 == 0 && a.gate_stride % 4 == 0 && a.out_stride % 4 == 0 && ptr_aligned(a.o, four) &&
                     ptr_aligned(a.gate, four) && ptr_aligned(a.out, four) && ptr_aligned(a.norm, 16);
    const dim3 grid((unsigned)rows), block(kThreads);
    if (per_head) {
#define GO(N) hipLaunchKernelGGL((decay_out_heads_kernel<T, N>), grid, block, 0, st, a)
        if (vec && a.vdim == 32) GO(8);
        else if (vec && a.vdim == 64) GO(16);
        else if (vec && a.vdim == 128) GO(32);
        else if (vec && a.vdim == 256) GO(64);
        else GO(0);
#undef GO
        return (int)hipGetLastError();
    }
    const int chunks = ((vec ? n / 4 : n) + kThreads - 1) / kThreads;
#define GO(V, N) hipLaunchKernelGGL((decay_out_row_kernel<T, V, N>), grid, block, 0, st, a)
    if (vec) {
        if (chunks <= 1) GO(4, 1);
        else if (chunks <= 2) GO(4, 2);
        else if (chunks <= 4) GO(4, 4);
        else if (chunks <= 8) GO(4, 8);
        else if (chunks <= 16) GO(4, 16);
        else return INFER_KV_EUNSUPPORTED;
    } else {
        if (chunks <= 4) GO(1, 4);
        else if (chunks <= 64) GO(1, 64);
        else return INFER_KV_EUNSUPPORTED;
    }
#undef GO
    return (int)hipGetLastError();
}

template <class T>
int launch_any(const DecayArgs<T>& a, const Span* spans, const int32_t* slots, const int64_t* positions, int64_t items, hipStream_t st) {
    if (items > 65535) return INFER_KV_EUNSUPPORTED;
    const size_t lds = (size_t)(a.dim_pad * 18 + 64) * sizeof(float);
    hipLaunchKernelGGL((decay_scan_any_kernel<T>), dim3((unsigned)(a.vdim_pad / 16), (unsigned)a.heads, (unsigned)items), dim3(kThreads), lds,
                       st, a, spans, slots, positions);
    return (int)hipGetLastError();
}

template <class T, bool FUSED>
int launch_step(const DecayArgs<T>& a, const DecayOutArgs<T>& b, const int32_t* slots, const int64_t* positions, int64_t rows, hipStream_t st) {
    const int cgs = a.vdim_pad / 4, rgs = kThreads / cgs, np = (a.dim_pad + rgs - 1) / rgs;
    const size_t lds = (size_t)(2 * a.dim_pad + a.vdim_pad + rgs * a.vdim_pad + 4) * sizeof(float);
    const dim3 grid((unsigned)rows, (unsigned)a.heads), block(kThreads);
#define GO(N) hipLaunchKernelGGL((decay_step_kernel<T, N, FUSED>), grid, block, lds, st, a, b, slots, positions)
    if (np <= 1) GO(1);
    else if (np <= 2) GO(2);
    else if (np <= 4) GO(4);
    else if (np <= 8) GO(8);
    else if (np <= 16) GO(16);
    else GO(32);
#undef GO
    return (int)hipGetLastError();
}

bool size_in(int64_t v, int64_t lo, int64_t hi) { return v >= lo && v <= hi; }

}  // namespace

// [0]: state rows per head, [1]: state columns per head; 0 if the sizes are served, otherwise a negative code
extern "C" int infer_decay_layout(int64_t dim, int64_t vdim, int64_t* out2) {
    if (!out2 || dim < 1 || vdim < 1) return INFER_KV_EINVAL;
    if (dim > 512 || vdim > 512) return INFER_KV_EUNSUPPORTED;
    out2[0] = (dim + 31) / 32 * 32;
    out2[1] = (vdim + 31) / 32 * 32;
    return INFER_KV_OK;
}

extern "C" int infer_decay_attention(int elem, const void* proj, int64_t proj_stride, int64_t q_off, int64_t k_off, int64_t v_off,
                                     int64_t g_off, int64_t heads, int64_t dim, int64_t vdim, const float* decay, int silu,
                                     const float* table, int64_t rot_dims, int64_t max_pos, float scale, const float* norm,
                                     int norm_per_head, int gate_silu, float eps, float* state, int64_t num_slots,
                                     const int32_t* slots, const int64_t* positions, int64_t decode_rows, const int32_t* spans,
                                     int64_t num_spans, int64_t rows, void* out, int64_t out_stride, void* stream) {
    int64_t pad[2];
    if (!size_in(rows, 0, 0x7fffffff) || !size_in(decode_rows, 0, rows) || !size_in(num_spans, 0, 65535)) return INFER_KV_EINVAL;
    if (rows == 0) return INFER_KV_OK;
    if (!proj || !decay || !state || !out || (decode_rows > 0 && (!slots || !positions)) || (decode_rows < rows && (!spans || num_spans < 1)))
        return INFER_KV_EINVAL;
    int rc = infer_decay_layout(dim, vdim, pad);
    if (rc) return rc;
    if (!size_in(heads, 1, 65535) || !size_in(num_slots, 1, 1 << 24) || !size_in(q_off, 0, proj_stride - heads * dim) ||
        !size_in(k_off, 0, proj_stride - heads * dim) || !size_in(v_off, 0, proj_stride - heads * vdim) ||
        !size_in(g_off, 0, proj_stride - heads * vdim) || out_stride < heads * vdim || rot_dims < 0 || rot_dims % 2 || rot_dims > dim ||
        (rot_dims > 0 && (!table || max_pos < 1)) || (silu && rot_dims > 0))
        return INFER_KV_EINVAL;
    if (!ptr_aligned(state, 16)) return INFER_KV_EALIGN;
    hipStream_t st = (hipStream_t)stream;
    auto go = [&](auto zero) {
        using T = decltype(zero);
        const T* p = (const T*)proj;
        DecayArgs<T> a{p, proj_stride, (int)q_off, (int)k_off, (int)v_off, (int)heads, (int)dim, (int)vdim, (int)pad[0], (int)pad[1], decay,
                       silu != 0, table, (int)(rot_dims / 2), rot_dims > 0 ? max_pos : 1, scale, state, (int)num_slots, (T*)out, out_stride};
        DecayOutArgs<T> b{(const T*)out, out_stride, p + g_off, proj_stride, norm, gate_silu != 0, (int)heads, (int)vdim, eps, (T*)out, out_stride};
        int64_t finished = 0;                                  // rows in front that are already normed and gated
        int rc = INFER_KV_OK;
        if (decode_rows > 0) {
            const int rgs = kThreads / (int)(pad[1] / 4);
            if ((pad[0] + rgs - 1) / rgs > 32) {
                rc = launch_any(a, nullptr, slots, positions, decode_rows, st);
            } else if (norm_per_head) {
                rc = launch_step<T, true>(a, b, slots, positions, decode_rows, st);
                finished = decode_rows;
            } else {
                rc = launch_step<T, false>(a, b, slots, positions, decode_rows, st);
            }
            if (rc) return rc;
        }
        if (decode_rows < rows) rc = launch_any(a, (const Span*)spans, nullptr, nullptr, num_spans, st);
        if (rc || finished == rows) return rc;
        b.o += finished * out_stride;
        b.out += finished * out_stride;
        b.gate += finished * proj_stride;
        return launch_out(b, norm_per_head != 0, rows - finished, st);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}
