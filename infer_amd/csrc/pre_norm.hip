// Float32 residual stream of a pre-norm decoder with a learned scale behind every sublayer, for gfx950 (MI355X).
//
//   pre_norm_kernel   x <- x + y * scale [+ first] [+ step] ;  h <- rms(x) * w
//                     in one pass over a row.  y is a sublayer's output: a tensor, the unreduced pieces of a split-K
//                     product, and/or the weighted sum of what a token's experts gave (moe.hip).  The sum can be the
//                     embedding lookup instead, with a second table that is addressed by a token and its predecessor.
//                     `first` (the embedding) and `step` (a vector) enter where a repeated run of layers starts.
//   softcap_kernel    logits <- cap * tanh(scale * logits / cap)
//
// HBM / latency bound: a row is read once, held in registers and written once.
#include "elem.h"

namespace {

constexpr int kThreads = 256;

template <class T>
struct PreNormArgs {
    const int64_t* tokens; const T* embed; int vocab;             // embedding lookup instead of the sum (x is only written)
    const int64_t* prev; const T* bigram; int64_t buckets, mul_prev, mul_cur;   // prev < 0: no predecessor, row `buckets`
    const T* y; int64_t y_stride;
    const float* partial; int splits; int64_t split_stride, partial_stride;
    const T* experts; const int32_t* places; const float* weights; int top;     // [place][width], [row][top]; place -1: h_in
    int64_t num_places;
    const T* h_in; int64_t h_in_stride;
    const float* scale;                                           // [width] or nullptr: 1
    float* first; bool write_first;                               // [row][width]: written with the lookup, otherwise added
    const float* step;                                            // [width]
    float* x; int64_t x_stride;
    const float* w;
    T* h; int64_t h_stride;
    int width;
    float eps;
};

template <int VEC, class T>
__device__ __forceinline__ void add_elems(const T* p, float f, float (&y)[VEC]) {
    float v[VEC];
    load_elems<VEC>(p, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) y[e] += f * v[e];
}

template <class T, int VEC, int NCH>
__global__ void __launch_bounds__(kThreads) pre_norm_kernel(PreNormArgs<T> a) {
    const int64_t row = blockIdx.x;
    const int tid = threadIdx.x;
    __shared__ float part[kThreads / 64];
    float* xr = a.x + row * a.x_stride;
    float x[NCH][VEC];
    auto col = [&](int j) { return (tid + j * kThreads) * VEC; };

    if (a.tokens) {
        int64_t tok = a.tokens[row];
        const int64_t before = a.bigram ? a.prev[row] : -1;
        const int64_t pair = before < 0 ? a.buckets : (before * a.mul_prev + tok * a.mul_cur) % (a.buckets > 0 ? a.buckets : 1);
        tok = tok < 0 ? 0 : (tok >= a.vocab ? a.vocab - 1 : tok);
#pragma unroll
        for (int j = 0; j < NCH; ++j) {
            const int c = col(j);
            if (c >= a.width) continue;
            load_elems<VEC>(a.embed + tok * a.width + c, x[j]);
            if (a.bigram) add_elems<VEC>(a.bigram + (pair < 0 ? 0 : pair) * a.width + c, 1.f, x[j]);
            if (a.write_first) store_elems<VEC>(a.first + row * a.width + c, x[j]);
        }
    } else {
        float y[NCH][VEC];
#pragma unroll
        for (int j = 0; j < NCH; ++j) {
            const int c = col(j);
            if (c >= a.width) continue;
            load_elems<VEC>(xr + c, x[j]);
#pragma unroll
            for (int e = 0; e < VEC; ++e) y[j][e] = 0.f;
            if (a.y) load_elems<VEC>(a.y + row * a.y_stride + c, y[j]);
            for (int s = 0; s < a.splits; ++s) add_elems<VEC>(a.partial + row * a.partial_stride + s * a.split_stride + c, 1.f, y[j]);
        }
        for (int k = 0; k < a.top; ++k) {
            const int64_t place = a.places[row * a.top + k];
            const float f = a.weights[row * a.top + k];
            const T* from = place < 0 || place >= a.num_places ? a.h_in + row * a.h_in_stride : a.experts + place * a.width;
#pragma unroll
            for (int j = 0; j < NCH; ++j)
                if (col(j) < a.width) add_elems<VEC>(from + col(j), f, y[j]);
        }
#pragma unroll
        for (int j = 0; j < NCH; ++j) {
            const int c = col(j);
            if (c >= a.width) continue;
            if (a.scale) {
                float s[VEC];
                load_elems<VEC>(a.scale + c, s);
#pragma unroll
                for (int e = 0; e < VEC; ++e) y[j][e] *= s[e];
            }
#pragma unroll
            for (int e = 0; e < VEC; ++e) x[j][e] += y[j][e];
            if (a.first) add_elems<VEC>(a.first + row * a.width + c, 1.f, x[j]);
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
        const int c = col(j);
        if (c >= a.width) continue;
        if (a.step) add_elems<VEC>(a.step + c, 1.f, x[j]);
        store_elems<VEC>(xr + c, x[j]);
#pragma unroll
        for (int e = 0; e < VEC; ++e) ss += x[j][e] * x[j][e];
    }
    const float rs = rsqrtf(block_sum<kThreads / 64>(ss, part) / (float)a.width + a.eps);
    T* hr = a.h + row * a.h_stride;
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
        const int c = col(j);
        if (c >= a.width) continue;
        float w[VEC], h[VEC];
        load_elems<VEC>(a.w + c, w);
#pragma unroll
        for (int e = 0; e < VEC; ++e) h[e] = x[j][e] * rs * w[e];
        store_elems<VEC>(hr + c, h);
    }
}

template <class T>
int launch_pre_norm(const PreNormArgs<T>& a, int64_t rows, hipStream_t stream) {
    const bool vec = a.width % 4 == 0 && a.x_stride % 4 == 0 && a.y_stride % 4 == 0 && a.h_stride % 4 == 0 && a.h_in_stride % 4 == 0 &&
                     a.partial_stride % 4 == 0 && a.split_stride % 4 == 0 && ptr_aligned(a.embed, 16) && ptr_aligned(a.bigram, 16) &&
                     ptr_aligned(a.y, 16) && ptr_aligned(a.partial, 16) && ptr_aligned(a.experts, 16) && ptr_aligned(a.h_in, 16) &&
                     ptr_aligned(a.scale, 16) && ptr_aligned(a.first, 16) && ptr_aligned(a.step, 16) && ptr_aligned(a.x, 16) &&
                     ptr_aligned(a.w, 16) && ptr_aligned(a.h, 16);
    const int units = vec ? a.width / 4 : a.width;
    const int chunks = (units + kThreads - 1) / kThreads;
    const dim3 grid((unsigned)rows), block(kThreads);
#define GO(V, N) hipLaunchKernelGGL((pre_norm_kernel<T, V, N>), grid, block, 0, stream, a)
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
__global__ void __launch_bounds__(256) softcap_kernel(const T* x, int64_t x_stride, float* out, int64_t cols, float cap, float factor) {
    const int64_t row = blockIdx.y;
    for (int64_t c = (int64_t)blockIdx.x * 256 + threadIdx.x; c < cols; c += (int64_t)gridDim.x * 256)
        out[row * cols + c] = cap * tanhf((float)x[row * x_stride + c] * factor);
}

}  // namespace

extern "C" int infer_pre_norm(int elem, const int64_t* tokens, const void* embed, int64_t vocab, const int64_t* prev,
                              const void* bigram, int64_t buckets, int64_t mul_prev, int64_t mul_cur, const void* y,
                              int64_t y_stride, const float* partial, int64_t splits, int64_t split_stride, int64_t partial_stride,
                              const void* experts, const int32_t* places, const float* weights, int64_t top, int64_t num_places,
                              const void* h_in, int64_t h_in_stride, const float* scale, float* first, const float* step, float* x,
                              int64_t x_stride, const float* w, void* h, int64_t h_stride, int64_t n_rows, int64_t width, float eps,
                              void* stream) {
    if (n_rows < 0 || width <= 0 || n_rows > 0x7fffffff || width > (1 << 20)) return INFER_KV_EINVAL;
    if (n_rows == 0) return INFER_KV_OK;
    if (!x || x_stride < width || !w || !h || h_stride < width) return INFER_KV_EINVAL;
    if (tokens && (!embed || vocab <= 0)) return INFER_KV_EINVAL;
    if (tokens && bigram && (!prev || buckets <= 0)) return INFER_KV_EINVAL;
    if (y && (y_stride < width || partial)) return INFER_KV_EINVAL;
    if (partial && (splits <= 0 || splits > 64 || partial_stride < width)) return INFER_KV_EINVAL;
    if (top < 0 || (top > 0 && (!places || !weights || !h_in || h_in_stride < width || num_places < 0 || (num_places > 0 && !experts))))
        return INFER_KV_EINVAL;
    if (!y) y_stride = 0;
    if (!partial) splits = split_stride = partial_stride = 0;
    if (top == 0) h_in_stride = 0;
    auto go = [&](auto zero) {
        using T = decltype(zero);
        const PreNormArgs<T> a{tokens, (const T*)embed, (int)vocab, prev, (const T*)bigram, buckets, mul_prev, mul_cur, (const T*)y, y_stride,
                               partial, (int)splits, split_stride, partial_stride, (const T*)experts, places, weights, (int)top, num_places,
                               (const T*)h_in, h_in_stride, scale, first, tokens != nullptr && first != nullptr, step, x, x_stride, w, (T*)h,
                               h_stride, (int)width, eps};
        return launch_pre_norm<T>(a, n_rows, (hipStream_t)stream);
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}

extern "C" int infer_softcap(int elem, const void* x, int64_t x_stride, float* out, int64_t n_rows, int64_t cols, float cap,
                             float scale, void* stream) {
    if (n_rows < 0 || cols <= 0 || !(cap > 0.f) || n_rows > 65535) return INFER_KV_EINVAL;
    if (n_rows == 0) return INFER_KV_OK;
    if (!x || !out || x_stride < cols) return INFER_KV_EINVAL;
    const int64_t blocks = (cols + 1023) / 1024;
    const dim3 grid((unsigned)(blocks < 4096 ? blocks : 4096), (unsigned)n_rows), block(256);
    if (elem == INFER_ELEM_BF16)
        hipLaunchKernelGGL((softcap_kernel<__bf16>), grid, block, 0, (hipStream_t)stream, (const __bf16*)x, x_stride, out, cols, cap, scale / cap);
    else if (elem == INFER_ELEM_F32)
        hipLaunchKernelGGL((softcap_kernel<float>), grid, block, 0, (hipStream_t)stream, (const float*)x, x_stride, out, cols, cap, scale / cap);
    else
        return INFER_KV_EUNSUPPORTED;
    return (int)hipGetLastError();
}
