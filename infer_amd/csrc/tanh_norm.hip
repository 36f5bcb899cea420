// Elementwise steps of a pre-norm decoder whose norm is a squashing function, for gfx950 (MI355X).
//
//   tanh_norm_kernel   x <- x + y [+ bias] ;  h <- tanh(alpha x) * w + b
//                      on the float32 residual stream.  y is a sublayer's output: a tensor or the unreduced pieces of a split-K
//                      product.  The sum can be the embedding lookup instead, x <- tanh(alpha' (embed * scale)) * w' + b'.
//   xielu_kernel       h <- act(x + bias) with the trainable activation
//                      act(z) = p z^2 + z / 2 for z > 0, q (e^z - 1 - z) + z / 2 otherwise
//
// HBM / latency bound, and free of reductions: a thread owns eight columns of a few consecutive rows and keeps what belongs to
// the columns in registers.
#include "elem.h"

namespace {

constexpr int kThreads = 256;

// e^z - 1 - z for z <= 0; the difference is a series where it would cancel
__device__ __forceinline__ float exp_rest_f(float z) {
    const float far = __builtin_amdgcn_exp2f(z * kLog2e) - 1.f - z;
    const float s = 1.f / 2 + z * (1.f / 6 + z * (1.f / 24 + z * (1.f / 120 + z * (1.f / 720 + z * (1.f / 5040)))));
    return z > -0.5f ? z * z * s : far;
}
// tanh z = 1 - 2 / (1 + e^2z); its Taylor series where that would cancel
__device__ __forceinline__ float tanh_f(float z) {
    const float y = z * z, a = fabsf(z);
    const float near = z + z * y * (-1.f / 3 + y * (2.f / 15 + y * (-17.f / 315 + y * (62.f / 2835 - y * (1382.f / 155925)))));
    const float far = 1.f - 2.f * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(2.f * kLog2e * a));
    return a < 0.3f ? near : copysignf(far, z);
}

template <class T>
struct TanhNormArgs {
    const int64_t* tokens; const T* embed; int vocab;             // embedding lookup instead of the sum (x is only written)
    float embed_scale, in_alpha; const float* in_w; const float* in_b;
    const T* y; int64_t y_stride;
    const float* partial; int splits; int64_t split_stride, partial_stride;
    const float* bias;                                            // [width] or nullptr
    float* x; int64_t x_stride;
    float alpha; const float* w; const float* b;
    T* h; int64_t h_stride;
    int64_t rows;
    int width;
};

// VEC columns and up to ROWS rows per thread
template <class T, int VEC, int ROWS>
__global__ void __launch_bounds__(kThreads) tanh_norm_kernel(TanhNormArgs<T> a) {
    const int c = (blockIdx.y * kThreads + threadIdx.x) * VEC;
    if (c >= a.width) return;
    const int64_t row0 = (int64_t)blockIdx.x * ROWS;
    float x[ROWS][VEC], y[ROWS][VEC], w[VEC], b[VEC], bias[VEC];
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {                              // everything is requested before anything is used
        const int64_t row = row0 + r < a.rows ? row0 + r : a.rows - 1;
        if (a.tokens) {
            int64_t tok = a.tokens[row];
            tok = tok < 0 ? 0 : (tok >= a.vocab ? a.vocab - 1 : tok);
            load_elems<VEC>(a.embed + tok * a.width + c, y[r]);
        } else {
            load_elems<VEC>(a.x + row * a.x_stride + c, x[r]);
            if (a.y) load_elems<VEC>(a.y + row * a.y_stride + c, y[r]);
        }
    }
    load_elems<VEC>(a.w + c, w);
    load_elems<VEC>(a.b + c, b);
#pragma unroll
    for (int e = 0; e < VEC; ++e) bias[e] = 0.f;
    if (a.bias) load_elems<VEC>(a.bias + c, bias);
    float in_w[VEC], in_b[VEC];
    if (a.tokens) {
        load_elems<VEC>(a.in_w + c, in_w);
        load_elems<VEC>(a.in_b + c, in_b);
    }
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
        const int64_t row = row0 + r;
        if (row >= a.rows) return;
        if (a.tokens) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) x[r][e] = tanh_f(a.in_alpha * (y[r][e] * a.embed_scale)) * in_w[e] + in_b[e];
        } else {
            if (a.partial) {
#pragma unroll
                for (int e = 0; e < VEC; ++e) y[r][e] = 0.f;
                for (int s = 0; s < a.splits; ++s) {
                    float v[VEC];
                    load_elems<VEC>(a.partial + row * a.partial_stride + s * a.split_stride + c, v);
#pragma unroll
                    for (int e = 0; e < VEC; ++e) y[r][e] += v[e];
                }
            }
#pragma unroll
            for (int e = 0; e < VEC; ++e) x[r][e] += y[r][e] + bias[e];
        }
        store_elems<VEC>(a.x + row * a.x_stride + c, x[r]);
        float h[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) h[e] = tanh_f(a.alpha * x[r][e]) * w[e] + b[e];
        store_elems<VEC>(a.h + row * a.h_stride + c, h);
    }
}

template <class T>
int launch_tanh_norm(const TanhNormArgs<T>& a, hipStream_t stream) {
    const bool vec = a.width % 8 == 0 && a.x_stride % 8 == 0 && a.y_stride % 8 == 0 && a.h_stride % 8 == 0 && a.partial_stride % 4 == 0 &&
                     a.split_stride % 4 == 0 && ptr_aligned(a.embed, 16) && ptr_aligned(a.in_w, 16) && ptr_aligned(a.in_b, 16) &&
                     ptr_aligned(a.y, 16) && ptr_aligned(a.partial, 16) && ptr_aligned(a.bias, 16) && ptr_aligned(a.x, 16) &&
                     ptr_aligned(a.w, 16) && ptr_aligned(a.b, 16) && ptr_aligned(a.h, 16);
    const int units = vec ? a.width / 8 : a.width;
    const unsigned cols = (unsigned)((units + kThreads - 1) / kThreads);
    if (cols > 65535) return INFER_KV_EUNSUPPORTED;
#define GO(V, R) hipLaunchKernelGGL((tanh_norm_kernel<T, V, R>), dim3((unsigned)((a.rows + R - 1) / R), cols), dim3(kThreads), 0, stream, a)
    if (!vec) GO(1, 1);
    else if (a.rows * cols >= 8192) GO(8, 4);                     // enough rows for everybody
    else GO(8, 1);
#undef GO
    return (int)hipGetLastError();
}

template <class T>
struct XieluArgs {
    const T* x; int64_t x_stride;
    const float* bias;
    float p, q;
    T* out; int64_t out_stride;
    int64_t rows;
    int cols;
};

template <class T, int VEC, int ROWS>
__global__ void __launch_bounds__(kThreads) xielu_kernel(XieluArgs<T> a) {
    const int c = (blockIdx.y * kThreads + threadIdx.x) * VEC;
    if (c >= a.cols) return;
    const int64_t row0 = (int64_t)blockIdx.x * ROWS;
    float x[ROWS][VEC], bias[VEC];
#pragma unroll
    for (int r = 0; r < ROWS; ++r) load_elems<VEC>(a.x + (row0 + r < a.rows ? row0 + r : a.rows - 1) * a.x_stride + c, x[r]);
    load_elems<VEC>(a.bias + c, bias);
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
        if (row0 + r >= a.rows) return;
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
            const float z = x[r][e] + bias[e];
            x[r][e] = (z > 0.f ? a.p * z * z : a.q * exp_rest_f(z)) + 0.5f * z;
        }
        store_elems<VEC>(a.out + (row0 + r) * a.out_stride + c, x[r]);
    }
}

template <class T>
int launch_xielu(const XieluArgs<T>& a, hipStream_t stream) {
    const bool vec = a.cols % 8 == 0 && a.x_stride % 8 == 0 && a.out_stride % 8 == 0 && ptr_aligned(a.x, 16) && ptr_aligned(a.bias, 16) &&
                     ptr_aligned(a.out, 16);
    const int units = vec ? a.cols / 8 : a.cols;
    const unsigned cols = (unsigned)((units + kThreads - 1) / kThreads);
    if (cols > 65535) return INFER_KV_EUNSUPPORTED;
#define GO(V, R) hipLaunchKernelGGL((xielu_kernel<T, V, R>), dim3((unsigned)((a.rows + R - 1) / R), cols), dim3(kThreads), 0, stream, a)
    if (!vec) GO(1, 1);
    else if (a.rows * cols >= 8192) GO(8, 4);
    else GO(8, 1);
#undef GO
    return (int)hipGetLastError();
}

}  // namespace

extern "C" int infer_tanh_norm(int elem, const int64_t* tokens, const void* embed, int64_t vocab, float embed_scale, float in_alpha,
                               const float* in_w, const float* in_b, const void* y, int64_t y_stride, const float* partial,
                               int64_t splits, int64_t split_stride, int64_t partial_stride, const float* bias, float* x,
                               int64_t x_stride, float alpha, const float* w, const float* b, void* h, int64_t h_stride,
                               int64_t n_rows, int64_t width, void* stream) {
    if (n_rows < 0 || width <= 0 || n_rows > 0x7fffffff || width > (1 << 20)) return INFER_KV_EINVAL;
    if (n_rows == 0) return INFER_KV_OK;
    if (!x || x_stride < width || !w || !b || !h || h_stride < width) return INFER_KV_EINVAL;
    if (tokens && (!embed || vocab <= 0 || !in_w || !in_b)) return INFER_KV_EINVAL;
    if (!tokens && !y == !partial) return INFER_KV_EINVAL;
    if (y && y_stride < width) return INFER_KV_EINVAL;
    if (partial && (splits <= 0 || splits > 64 || partial_stride < width)) return INFER_KV_EINVAL;
    if (!y) y_stride = 0;
    if (!partial) splits = split_stride = partial_stride = 0;
    auto go = [&](auto zero) {
        using T = decltype(zero);
        const TanhNormArgs<T> a{tokens, (const T*)embed, (int)vocab, embed_scale, in_alpha, in_w, in_b, (const T*)y, y_stride, partial,
                                (int)splits, split_stride, partial_stride, bias, x, x_stride, alpha, w, b, (T*)h, h_stride, n_rows, (int)width};
        return launch_tanh_norm<T>(a, (hipStream_t)stream);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}

extern "C" int infer_xielu(int elem, const void* x, int64_t x_stride, const float* bias, float p, float q, void* out, int64_t out_stride,
                           int64_t n_rows, int64_t cols, void* stream) {
    if (n_rows < 0 || cols <= 0 || n_rows > 0x7fffffff || cols > (1 << 24)) return INFER_KV_EINVAL;
    if (n_rows == 0) return INFER_KV_OK;
    if (!x || x_stride < cols || !bias || !out || out_stride < cols) return INFER_KV_EINVAL;
    auto go = [&](auto zero) {
        using T = decltype(zero);
        return launch_xielu<T>(XieluArgs<T>{(const T*)x, x_stride, bias, p, q, (T*)out, out_stride, n_rows, (int)cols}, (hipStream_t)stream);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}
