// Residual stream in float32 with a norm on both sides of every sublayer, and the gated activation of its
// feed-forward, for gfx950 (MI355X).
//
//   residual_norm_kernel   x <- x + rms(y) * w_post ;  h <- rms(x) * w_pre
//                          in one pass over a row: the norm behind a sublayer, the residual sum and the
//                          norm in front of the next sublayer.  Either half can be left out, the first can
//                          be the embedding lookup instead, and y can be the unreduced partial sums of the
//                          split-K GEMM (skinny_gemm.hip).
//                          POST: the norm behind the residual sum instead,
//                          x <- rms(alpha * x + y) * w_post ;  h <- x, or rms(x) * w_pre behind the last sublayer
//   gated_act_kernel       h <- act(g) * u with act = gelu_tanh or silu, or a clamped gate
//
// HBM / latency bound: a row is read once, held in registers between the reductions and written once.
#include "elem.h"

namespace {

constexpr int kThreads = 256;

template <class T>
struct ResidualNormArgs {
    const int64_t* tokens;        // embedding lookup instead of the residual (x is only written)
    const T* embed;
    float embed_scale;
    int vocab;
    const T* y; int64_t y_stride;                 // sublayer output, or
    const float* partial; int splits; int64_t split_stride; int64_t partial_stride;   // its split-K pieces
    const float* w_post;
    float* x; int64_t x_stride;
    const float* w_pre;
    T* h; int64_t h_stride;
    int width;
    float eps;
    float alpha;                                  // POST
};

template <class T, int VEC, int NCH, bool POST>
__global__ void __launch_bounds__(kThreads) residual_norm_kernel(ResidualNormArgs<T> a) {
    const int64_t row = blockIdx.x;
    const int tid = threadIdx.x;
    __shared__ float part[2][kThreads / 64];
    float* xr = a.x + row * a.x_stride;
    float x[NCH][VEC];
    const bool has_y = a.y != nullptr || a.partial != nullptr;

    if (a.tokens) {
        int64_t tok = a.tokens[row];
        tok = tok < 0 ? 0 : (tok >= a.vocab ? a.vocab - 1 : tok);
        const T* er = a.embed + tok * a.width;
#pragma unroll
        for (int j = 0; j < NCH; ++j) {
            const int c = (tid + j * kThreads) * VEC;
            if (c < a.width) {
                load_elems<VEC>(er + c, x[j]);
#pragma unroll
                for (int e = 0; e < VEC; ++e) x[j][e] *= a.embed_scale;
            }
        }
    } else {
#pragma unroll
        for (int j = 0; j < NCH; ++j) {
            const int c = (tid + j * kThreads) * VEC;
            if (c < a.width) load_elems<VEC>(xr + c, x[j]);
        }
    }
    if (has_y) {
        float y[NCH][VEC];
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < NCH; ++j) {
            const int c = (tid + j * kThreads) * VEC;
            if (c < a.width) {
                if (a.partial) {
#pragma unroll
                    for (int e = 0; e < VEC; ++e) y[j][e] = 0.f;
                    const float* pp = a.partial + row * a.partial_stride + c;
                    for (int s = 0; s < a.splits; ++s) {
                        float v[VEC];
                        load_elems<VEC>(pp + s * a.split_stride, v);
#pragma unroll
                        for (int e = 0; e < VEC; ++e) y[j][e] += v[e];
                    }
                } else {
                    load_elems<VEC>(a.y + row * a.y_stride + c, y[j]);
                }
#pragma unroll
                for (int e = 0; e < VEC; ++e) {
                    if constexpr (POST) y[j][e] += a.alpha * x[j][e];
                    ss += y[j][e] * y[j][e];
                }
            }
        }
        const float rs = rsqrtf(block_sum<kThreads / 64>(ss, part[0]) / (float)a.width + a.eps);
#pragma unroll
        for (int j = 0; j < NCH; ++j) {
            const int c = (tid + j * kThreads) * VEC;
            if (c < a.width) {
                float w[VEC];
                load_elems<VEC>(a.w_post + c, w);
#pragma unroll
                for (int e = 0; e < VEC; ++e) {
                    const float v = y[j][e] * rs * w[e];
                    x[j][e] = POST ? v : x[j][e] + v;
                }
            }
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
        const int c = (tid + j * kThreads) * VEC;
        if (c < a.width) {
            if (has_y || a.tokens) store_elems<VEC>(xr + c, x[j]);
#pragma unroll
            for (int e = 0; e < VEC; ++e) ss += x[j][e] * x[j][e];
        }
    }
    if (!a.w_pre) {
        if constexpr (POST) {
#pragma unroll
            for (int j = 0; j < NCH; ++j) {
                const int c = (tid + j * kThreads) * VEC;
                if (c < a.width) store_elems<VEC>(a.h + row * a.h_stride + c, x[j]);
            }
        }
        return;
    }
    const float rs = rsqrtf(block_sum<kThreads / 64>(ss, part[1]) / (float)a.width + a.eps);
    T* hr = a.h + row * a.h_stride;
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
        const int c = (tid + j * kThreads) * VEC;
        if (c < a.width) {
            float w[VEC], h[VEC];
            load_elems<VEC>(a.w_pre + c, w);
#pragma unroll
            for (int e = 0; e < VEC; ++e) h[e] = x[j][e] * rs * w[e];
            store_elems<VEC>(hr + c, h);
        }
    }
}

template <class T, bool POST>
int launch_residual_norm(const ResidualNormArgs<T>& a, int64_t rows, hipStream_t stream) {
    const bool vec = a.width % 4 == 0 && a.x_stride % 4 == 0 && a.y_stride % 4 == 0 && a.h_stride % 4 == 0 &&
                     a.partial_stride % 4 == 0 && a.split_stride % 4 == 0 && ptr_aligned(a.embed, 16) &&
                     ptr_aligned(a.y, 16) && ptr_aligned(a.partial, 16) && ptr_aligned(a.x, 16) && ptr_aligned(a.h, 16) &&
                     ptr_aligned(a.w_post, 16) && ptr_aligned(a.w_pre, 16);
    const int units = vec ? a.width / 4 : a.width;
    const int chunks = (units + kThreads - 1) / kThreads;
    const dim3 grid((unsigned)rows), block(kThreads);
#define GO(V, N) hipLaunchKernelGGL((residual_norm_kernel<T, V, N, POST>), grid, block, 0, stream, a)
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
struct GatedActArgs {
    T* out; int64_t out_stride;
    const T* x; int64_t x_stride;
    int d;
    int64_t total;      // rows * d / VEC
    float limit;        // kClamped
};

enum class Act { kGeluTanh, kSilu, kClamped };

// min(g, limit) sigmoid(1.702 min(g, limit)) (clamp(u, -limit, limit) + 1)
__device__ __forceinline__ float clamped_gate_f(float g, float u, float limit) {
    g = fminf(g, limit);
    return g * sigmoid_f(1.702f * g) * (fminf(fmaxf(u, -limit), limit) + 1.f);
}

template <class T, int VEC, Act ACT>
__global__ void __launch_bounds__(256) gated_act_kernel(GatedActArgs<T> a) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= a.total) return;
    const int per_row = a.d / VEC;
    const int64_t row = i / per_row;
    const int c = (int)(i - row * per_row) * VEC;
    float g[VEC], u[VEC];
    load_elems<VEC>(a.x + row * a.x_stride + c, g);
    load_elems<VEC>(a.x + row * a.x_stride + a.d + c, u);
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
        if constexpr (ACT == Act::kClamped) g[e] = clamped_gate_f(g[e], u[e], a.limit);
        else g[e] = (ACT == Act::kSilu ? silu_f(g[e]) : gelu_tanh_f(g[e])) * u[e];
    }
    store_elems<VEC>(a.out + row * a.out_stride + c, g);
}

template <class T, Act ACT>
int launch_gated_act(void* out, int64_t out_stride, const void* x, int64_t x_stride, int64_t rows, int64_t d,
                     float limit, hipStream_t stream) {
    const size_t bytes = 8 * sizeof(T) < 16 ? 8 * sizeof(T) : 16;
    const bool vec = d % 8 == 0 && out_stride % 8 == 0 && x_stride % 8 == 0 && ptr_aligned(out, bytes) && ptr_aligned(x, bytes);
    const int64_t total = rows * (vec ? d / 8 : d);
    const int64_t blocks = (total + 255) / 256;
    if (blocks > 0x7fffffff) return INFER_KV_EINVAL;
    GatedActArgs<T> a{(T*)out, out_stride, (const T*)x, x_stride, (int)d, total, limit};
    if (vec) hipLaunchKernelGGL((gated_act_kernel<T, 8, ACT>), dim3((unsigned)blocks), dim3(256), 0, stream, a);
    else hipLaunchKernelGGL((gated_act_kernel<T, 1, ACT>), dim3((unsigned)blocks), dim3(256), 0, stream, a);
    return (int)hipGetLastError();
}

template <Act ACT>
int gated_act(int elem, void* out, int64_t out_stride, const void* x, int64_t x_stride, int64_t n_rows, int64_t d, void* stream,
              float limit = 0.f) {
    if (n_rows < 0 || d <= 0 || d > (1 << 24)) return INFER_KV_EINVAL;
    if (n_rows == 0) return INFER_KV_OK;
    if (!out || !x || out_stride < d || x_stride < 2 * d) return INFER_KV_EINVAL;
    if (elem == INFER_ELEM_BF16) return launch_gated_act<__bf16, ACT>(out, out_stride, x, x_stride, n_rows, d, limit, (hipStream_t)stream);
    if (elem == INFER_ELEM_F32) return launch_gated_act<float, ACT>(out, out_stride, x, x_stride, n_rows, d, limit, (hipStream_t)stream);
    return INFER_KV_EUNSUPPORTED;
}

template <bool POST>
int residual_norm(int elem, const int64_t* tokens, const void* embed, float embed_scale, int64_t vocab, const void* y,
                  int64_t y_stride, const float* partial, int64_t splits, int64_t split_stride, int64_t partial_stride,
                  float alpha, const float* w_post, float* x, int64_t x_stride, const float* w_pre, void* h, int64_t h_stride,
                  int64_t n_rows, int64_t width, float eps, void* stream) {
    if (n_rows < 0 || width <= 0 || n_rows > 0x7fffffff || width > (1 << 20)) return INFER_KV_EINVAL;
    if (n_rows == 0) return INFER_KV_OK;
    const bool writes_h = POST || w_pre;
    if (!x || x_stride < width || (writes_h && (!h || h_stride < width))) return INFER_KV_EINVAL;
    if (tokens && (!embed || vocab <= 0)) return INFER_KV_EINVAL;
    if ((y || partial) && !w_post) return INFER_KV_EINVAL;
    if (y && (y_stride < width || partial)) return INFER_KV_EINVAL;
    if (partial && (splits <= 0 || splits > 64 || partial_stride < width)) return INFER_KV_EINVAL;
    if (!y) y_stride = 0;
    if (!partial) splits = split_stride = partial_stride = 0;
    if (!writes_h) { h = nullptr; h_stride = 0; }
    auto go = [&](auto zero) {
        using T = decltype(zero);
        const ResidualNormArgs<T> a{tokens, (const T*)embed, embed_scale, (int)vocab, (const T*)y, y_stride, partial, (int)splits,
                                    split_stride, partial_stride, w_post, x, x_stride, w_pre, (T*)h, h_stride, (int)width, eps, alpha};
        return launch_residual_norm<T, POST>(a, n_rows, (hipStream_t)stream);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}

}  // namespace

extern "C" int infer_residual_norm(int elem, const int64_t* tokens, const void* embed, float embed_scale, int64_t vocab,
                                   const void* y, int64_t y_stride, const float* partial, int64_t splits,
                                   int64_t split_stride, int64_t partial_stride, const float* w_post, float* x,
                                   int64_t x_stride, const float* w_pre, void* h, int64_t h_stride, int64_t n_rows,
                                   int64_t width, float eps, void* stream) {
    return residual_norm<false>(elem, tokens, embed, embed_scale, vocab, y, y_stride, partial, splits, split_stride, partial_stride,
                                1.f, w_post, x, x_stride, w_pre, h, h_stride, n_rows, width, eps, stream);
}

extern "C" int infer_post_norm(int elem, const int64_t* tokens, const void* embed, float embed_scale, int64_t vocab,
                               const void* y, int64_t y_stride, const float* partial, int64_t splits, int64_t split_stride,
                               int64_t partial_stride, float alpha, const float* w_post, float* x, int64_t x_stride,
                               const float* w_last, void* h, int64_t h_stride, int64_t n_rows, int64_t width, float eps,
                               void* stream) {
    return residual_norm<true>(elem, tokens, embed, embed_scale, vocab, y, y_stride, partial, splits, split_stride, partial_stride,
                               alpha, w_post, x, x_stride, w_last, h, h_stride, n_rows, width, eps, stream);
}

extern "C" int infer_gelu_tanh_and_mul(int elem, void* out, int64_t out_stride, const void* x, int64_t x_stride,
                                       int64_t n_rows, int64_t d, void* stream) {
    return gated_act<Act::kGeluTanh>(elem, out, out_stride, x, x_stride, n_rows, d, stream);
}

extern "C" int infer_silu_and_mul(int elem, void* out, int64_t out_stride, const void* x, int64_t x_stride,
                                  int64_t n_rows, int64_t d, void* stream) {
    return gated_act<Act::kSilu>(elem, out, out_stride, x, x_stride, n_rows, d, stream);
}

extern "C" int infer_clamped_gate_and_mul(int elem, void* out, int64_t out_stride, const void* x, int64_t x_stride,
                                          int64_t n_rows, int64_t d, float limit, void* stream) {
    return gated_act<Act::kClamped>(elem, out, out_stride, x, x_stride, n_rows, d, stream, limit);
}
