// Selective state space (Mamba-2: Dao and Gu, "Transformers are SSMs: Generalized Models and Efficient Algorithms Through
// Structured State Space Duality"), for gfx950 (MI355X).  Per head, over a float32 state S[state][vdim]:
//     S <- e^{a dt} S + dt B x^T ;   y = S^T C + D x ,   dt = softplus(. + bias), a = -e^{A_log}
// with x, B and C behind a causal convolution per channel and silu; groups of heads share B and C.  Behind it
// rms(y silu(z)) over equal parts of a token's channels.
//
//   ssm_step_kernel      one token per sequence (decode): convolution, step sizes and recurrence, one workgroup per
//                        (sequence, head), the state passes through registers once
//   ssm_conv_kernel      convolution and silu of prompt portions
//   ssm_chunk_kernel     prompt portions in chunks of 32 tokens on bf16 matrix instructions
//   ssm_join_kernel      carries the state over the segments that a long portion is cut into
//   ssm_scan_any_kernel  prompt portions of any size and element type, token by token
//   ssm_norm_kernel      gate and norm of all rows; keeps the last inputs of the convolution
//
// The convolution's inputs live in a ring of `taps` entries per slot (position mod taps), one more than it looks back, so a
// decode launch may write its entry while others read.  A sequence at position 0 starts from zeros whatever its slot holds.
//
// Chunk form.  With S the state before a chunk of n tokens and G the running sum of a dt,
//     y_i = e^{G_i} S^T C_i + sum_{j<=i} e^{G_i-G_j} dt_j (C_i B_j) x_j + D x_i ,   S' = e^{G_n} S + sum_j B_j (e^{G_n-G_j} dt_j x_j)^T .
// No exponent is positive.  x, B and C are bf16 already; the weighted x enters the state as three bf16 pieces (exact to
// float precision), the products of the output, which is rounded to bf16 next, take two (2^-17).
#include "elem.h"
#include "pieces.h"

namespace {

typedef short i16x4 __attribute__((ext_vector_type(4)));
typedef short i16x8 __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) i16x4 lds_i16x4;

constexpr int kThreads = 256;
constexpr int kC = 32;          // tokens per chunk
constexpr int kSlab = 64;       // state columns per workgroup of the chunk kernel
constexpr int kAhead = kThreads / 64;   // chunks whose step sizes are computed together, one per wavefront

struct Span { int32_t row0, count, slot, pos0; };       // consecutive tokens of one sequence

template <class T>
struct SsmArgs {
    const T* proj; int64_t proj_stride; int z_off, x_off, dt_off;   // [z: heads x vdim | x | B: groups x state | C | dt: heads]
    int heads, vdim, state_n, groups, channels, taps;
    const float* conv; const float* conv_bias;                      // [channels][taps] (last: the current token), [channels]
    const float* dt_bias; const float* a_log; const float* d;       // [heads]
    T* ring; float* state; int num_slots;                           // [slots][taps][channels], [slots][heads][state][vdim]
    T* y; int64_t y_stride;                                         // [row][heads * vdim]
    const T* xbc; int64_t xbc_stride; int64_t xbc_row0;             // rows from xbc_row0 on, behind convolution and silu
};

template <class T>
__device__ __forceinline__ float step_size(const SsmArgs<T>& a, int64_t row, int h) {
    return softplus_f((float)a.proj[row * a.proj_stride + a.dt_off + h] + a.dt_bias[h]);
}

// ------------------------------------------------------------------ decode
template <class T, int VEC>
__global__ void __launch_bounds__(kThreads) ssm_step_kernel(SsmArgs<T> a, const int32_t* slots, const int64_t* positions) {
    extern __shared__ float lds[];
    const int h = blockIdx.x, tid = threadIdx.x;
    const int64_t row = blockIdx.y;
    const int slot = slots[row];
    const int64_t pos = positions[row];
    const int n = a.state_n, inner = a.heads * a.vdim, per = a.heads / a.groups, grp = h / per;
    if (slot < 0 || slot >= a.num_slots) {               // padding
        for (int i = tid; i < a.vdim; i += kThreads) a.y[row * a.y_stride + h * a.vdim + i] = (T)0.f;
        return;
    }
    float* xs = lds;                                     // [vdim], then B and C [state] each, then the sums [rows][vdim]
    float* bs = xs + (a.vdim + 3) / 4 * 4;
    float* sums = bs + 2 * ((n + 3) / 4 * 4);
    float* cs = bs + (n + 3) / 4 * 4;
    const T* in = a.proj + row * a.proj_stride + a.x_off;
    T* ring = a.ring + (int64_t)slot * a.taps * a.channels;
    const int now = (int)(pos % a.taps);
    for (int i = tid; i < a.vdim + 2 * n; i += kThreads) {
        const int c = i < a.vdim ? h * a.vdim + i : i < a.vdim + n ? inner + grp * n + (i - a.vdim)
                                                                   : inner + (a.groups + grp) * n + (i - a.vdim - n);
        const T cur = in[c];
        float v = a.conv_bias[c] + (float)cur * a.conv[(int64_t)c * a.taps + a.taps - 1];
        int at = now;
        for (int k = 1; k < a.taps; ++k) {
            at = at == 0 ? a.taps - 1 : at - 1;
            if (pos >= k) v += (float)ring[(int64_t)at * a.channels + c] * a.conv[(int64_t)c * a.taps + a.taps - 1 - k];
        }
        if (i < a.vdim || h % per == 0) ring[(int64_t)now * a.channels + c] = cur;
        v = silu_f(v);
        if (i < a.vdim) xs[i] = v;
        else if (i < a.vdim + n) bs[i - a.vdim] = v;
        else cs[i - a.vdim - n] = v;
    }
    const float dt = step_size(a, row, h), decay = expf(-expf(a.a_log[h]) * dt);
    __syncthreads();
    const int quads = a.vdim / VEC, rows = kThreads / quads;
    const int q = tid % quads, r = tid / quads;
    float y[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) y[e] = 0.f;
    if (r < rows) {
        float* st = a.state + ((int64_t)slot * a.heads + h) * n * a.vdim + VEC * q;
        float dx[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) dx[e] = dt * xs[VEC * q + e];
        constexpr int kBatch = 8;
        for (int i0 = r; i0 < n; i0 += kBatch * rows) {
            float s[kBatch][VEC];
#pragma unroll
            for (int b = 0; b < kBatch; ++b) {
                const int i = i0 + b * rows;
#pragma unroll
                for (int e = 0; e < VEC; ++e) s[b][e] = 0.f;
                if (i < n && pos > 0) load_elems<VEC>(st + (int64_t)i * a.vdim, s[b]);
            }
#pragma unroll
            for (int b = 0; b < kBatch; ++b) {
                const int i = i0 + b * rows;
                if (i >= n) continue;
                const float bi = bs[i], ci = cs[i];
#pragma unroll
                for (int e = 0; e < VEC; ++e) {
                    s[b][e] = decay * s[b][e] + bi * dx[e];
                    y[e] += s[b][e] * ci;
                }
                store_elems<VEC>(st + (int64_t)i * a.vdim, s[b]);
            }
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) sums[r * a.vdim + VEC * q + e] = y[e];
    }
    __syncthreads();
    const float dh = a.d[h];
    for (int i = tid; i < a.vdim; i += kThreads) {
        float v = dh * xs[i];
        for (int k = 0; k < rows; ++k) v += sums[k * a.vdim + i];
        a.y[row * a.y_stride + h * a.vdim + i] = (T)v;
    }
}

// ------------------------------------------------------------------ convolution of portions
constexpr int kConvTokens = 16;         // per thread

// VEC channels per thread over 16 consecutive tokens; TAPS > 0: the inputs it looks back on stay in registers
template <class T, int VEC, int TAPS>
__global__ void __launch_bounds__(kThreads) ssm_conv_kernel(SsmArgs<T> a, const Span* spans, T* out) {
    const Span span = spans[blockIdx.z];
    const int c = (blockIdx.x * kThreads + threadIdx.x) * VEC, i0 = blockIdx.y * kConvTokens;
    if (c >= a.channels || i0 >= span.count || span.slot < 0 || span.slot >= a.num_slots) return;
    const T* in = a.proj + (int64_t)span.row0 * a.proj_stride + a.x_off + c;
    const T* ring = a.ring + (int64_t)span.slot * a.taps * a.channels + c;
    auto input = [&](int i, float (&x)[VEC]) {           // token i of the portion, in front of it if negative
        const int pos = span.pos0 + i;
        if (i >= 0) {
            load_elems<VEC>(in + (int64_t)i * a.proj_stride, x);
        } else if (pos >= 0) {
            load_elems<VEC>(ring + (int64_t)(pos % a.taps) * a.channels, x);
        } else {
#pragma unroll
            for (int e = 0; e < VEC; ++e) x[e] = 0.f;
        }
    };
    T* o = out + (span.row0 - a.xbc_row0 + i0) * a.xbc_stride + c;
    const int end = i0 + kConvTokens < span.count ? kConvTokens : span.count - i0;
    float bias[VEC];
    load_elems<VEC>(a.conv_bias + c, bias);
    if constexpr (TAPS > 0) {
        float w[TAPS][VEC], x[TAPS][VEC];
#pragma unroll
        for (int k = 0; k < TAPS; ++k)
#pragma unroll
            for (int e = 0; e < VEC; ++e) w[k][e] = a.conv[(int64_t)(c + e) * TAPS + k];
#pragma unroll
        for (int k = 0; k + 1 < TAPS; ++k) input(i0 + k - (TAPS - 1), x[k]);
        // inputs are requested in batches: the compiler moves no load in front of a store
        struct alignas(sizeof(T) * VEC < 16 ? sizeof(T) * VEC : 16) Raw { T e[VEC]; };
        constexpr int kBatch = 8;
#pragma unroll
        for (int b = 0; b < kConvTokens; b += kBatch) {
            if (b >= end) break;
            Raw raw[kBatch];
#pragma unroll
            for (int i = 0; i < kBatch; ++i)
                raw[i] = *reinterpret_cast<const Raw*>(in + (int64_t)(i0 + (b + i < end ? b + i : end - 1)) * a.proj_stride);
#pragma unroll
            for (int i = 0; i < kBatch; ++i) {
                float v[VEC];
#pragma unroll
                for (int e = 0; e < VEC; ++e) {
                    x[TAPS - 1][e] = (float)raw[i].e[e];
                    v[e] = bias[e];
#pragma unroll
                    for (int k = 0; k < TAPS; ++k) v[e] += w[k][e] * x[k][e];
                    v[e] = silu_f(v[e]);
                }
                if (b + i < end) store_elems<VEC>(o + (int64_t)(b + i) * a.xbc_stride, v);
#pragma unroll
                for (int k = 0; k + 1 < TAPS; ++k)
#pragma unroll
                    for (int e = 0; e < VEC; ++e) x[k][e] = x[k + 1][e];
            }
        }
    } else {
        for (int i = 0; i < end; ++i) {
            float v[VEC];
#pragma unroll
            for (int e = 0; e < VEC; ++e) v[e] = bias[e];
            for (int k = 0; k < a.taps; ++k) {
                float x[VEC];
                input(i0 + i + k - (a.taps - 1), x);
#pragma unroll
                for (int e = 0; e < VEC; ++e) v[e] += x[e] * a.conv[(int64_t)(c + e) * a.taps + k];
            }
#pragma unroll
            for (int e = 0; e < VEC; ++e) v[e] = silu_f(v[e]);
            store_elems<VEC>(o + (int64_t)i * a.xbc_stride, v);
        }
    }
}

// ------------------------------------------------------------------ any size
// One workgroup per (16 columns of the state, head, span); thread (r, c): column c, state rows r, r + 16, ...
template <class T, int NI>
__global__ void __launch_bounds__(kThreads) ssm_scan_any_kernel(SsmArgs<T> a, const Span* spans) {
    __shared__ float part[2][4][16];
    const Span span = spans[blockIdx.z];
    const int h = blockIdx.y, tid = threadIdx.x, r = tid >> 4, p = blockIdx.x * 16 + (tid & 15);
    if (span.slot < 0 || span.slot >= a.num_slots) return;
    const int n = a.state_n, inner = a.heads * a.vdim, grp = h / (a.heads / a.groups);
    const bool live = p < a.vdim;
    float* st = a.state + ((int64_t)span.slot * a.heads + h) * n * a.vdim + p;
    float s[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        const int k = r + 16 * i;
        s[i] = live && k < n && span.pos0 > 0 ? st[(int64_t)k * a.vdim] : 0.f;
    }
    const float ah = -expf(a.a_log[h]), dh = a.d[h];
    for (int t = 0; t < span.count; ++t) {
        const int64_t row = span.row0 + t;
        const T* in = a.xbc + (row - a.xbc_row0) * a.xbc_stride;
        const float dt = step_size(a, row, h), decay = expf(ah * dt);
        const float x = live ? (float)in[h * a.vdim + p] : 0.f;
        const T* b = in + inner + grp * n;
        const T* c = b + a.groups * n;
        float y = 0.f;
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            const int k = r + 16 * i;
            if (k < n) {
                s[i] = decay * s[i] + dt * (float)b[k] * x;
                y += s[i] * (float)c[k];
            }
        }
        y += __shfl_xor(y, 16, 64);
        y += __shfl_xor(y, 32, 64);
        if ((tid & 63) < 16) part[t & 1][tid >> 6][tid & 15] = y;
        __syncthreads();
        if (tid < 16 && live) {
            const float(*q)[16] = part[t & 1];
            a.y[row * a.y_stride + h * a.vdim + p] = (T)(q[0][tid] + q[1][tid] + q[2][tid] + q[3][tid] + dh * x);
        }
    }
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        const int k = r + 16 * i;
        if (live && k < n) st[(int64_t)k * a.vdim] = s[i];
    }
}

// ------------------------------------------------------------------ chunks
struct ChunkArgs {
    SsmArgs<__bf16> a;
    const Span* spans;
    int seg_len, max_seg, slabs;                 // tokens per segment (a multiple of kC), segments of the longest span
    float* ws;                                   // [span][max_seg][heads][state][vdim], then [span][max_seg][heads]: log2 of the decay
    float* ws_decay;
};

// A workgroup of four wavefronts serves one head and 64 columns of its state over the chunks of one segment; wavefront w owns 16
// columns as accumulators: lane (g, n) holds state rows 16 t + 4 g + e of column n.  That is an operand of the product with C as it
// lies, when the state rows of a k-step of 32 are taken in the order 16 tau + 4 g + e.  The 32 x 32 products C_i B_j are shared
// out over the wavefronts, weighted, and exchanged through LDS.  OUT = false: only the final state, from zero.
template <int NS, bool OUT>
__global__ void __launch_bounds__(kThreads, 2) ssm_chunk_kernel(ChunkArgs args) {
    constexpr int kRow = NS * 64 + 16, kXRow = 2 * kSlab + 16, kMRow = 2 * kC + 16;      // bytes
    constexpr int NU = NS > 2 ? NS / 2 : 1;                      // 16-byte units of B (and of C) per thread
    __shared__ __attribute__((aligned(16))) unsigned char bbuf[kC * kRow], cbuf[OUT ? kC * kRow : 16], xbuf[kC * kXRow];
    __shared__ __attribute__((aligned(16))) unsigned char mbuf[OUT ? 2 * kC * kMRow : 16];
    __shared__ __attribute__((aligned(16))) float sums[kAhead][kC], steps[kAhead][kC], weights[kAhead][kC];
    const SsmArgs<__bf16>& a = args.a;
    const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, n = lane & 15;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int h = blockIdx.y, slab = blockIdx.x % args.slabs, seg = blockIdx.x / args.slabs;
    const Span span = args.spans[blockIdx.z];
    const int first = seg * args.seg_len;
    if (span.slot < 0 || span.slot >= a.num_slots || first >= span.count) return;
    const bool last_seg = first + args.seg_len >= span.count;
    if (!OUT && last_seg) return;                                // nobody needs its final state yet
    const int count = last_seg ? span.count - first : args.seg_len;
    const int row0 = span.row0 + first, chunks = (count + kC - 1) / kC;
    const int N = a.state_n, inner = a.heads * a.vdim, grp = h / (a.heads / a.groups);
    const int v0 = slab * kSlab + wave * 16;                     // this wavefront's first column
    const int64_t state_len = (int64_t)N * a.vdim;
    float* from = a.state + ((int64_t)span.slot * a.heads + h) * state_len;
    float* to = from;
    const int64_t rec = ((int64_t)blockIdx.z * args.max_seg + seg) * a.heads + h;
    if (args.max_seg > 1) {
        if (OUT) from = args.ws + rec * state_len;
        else to = args.ws + rec * state_len;
    }
    const bool load = OUT && (args.max_seg > 1 || span.pos0 > 0), col_live = v0 + n < a.vdim;

    f32x4_t s[2 * NS];
#pragma unroll
    for (int t = 0; t < 2 * NS; ++t) {
        s[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        if (load && col_live)
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (16 * t + 4 * g + e < N) s[t][e] = from[(int64_t)(16 * t + 4 * g + e) * a.vdim + v0 + n];
    }
    // entries behind the real sizes stay zero
    for (int i = tid; i < (int)sizeof(bbuf) / 16; i += kThreads) reinterpret_cast<u32x4_t*>(bbuf)[i] = u32x4_t{0u, 0u, 0u, 0u};
    for (int i = tid; i < (int)sizeof(cbuf) / 16; i += kThreads) reinterpret_cast<u32x4_t*>(cbuf)[i] = u32x4_t{0u, 0u, 0u, 0u};
    for (int i = tid; i < (int)sizeof(xbuf) / 16; i += kThreads) reinterpret_cast<u32x4_t*>(xbuf)[i] = u32x4_t{0u, 0u, 0u, 0u};

    const int units = N / 8;
    int u_tok[NU], u_col[NU];                                    // token -1: no such unit; its load repeats another one
#pragma unroll
    for (int i = 0; i < NU; ++i) {
        const int u = tid + kThreads * i;
        u_tok[i] = u < kC * units ? u / units : -1;
        u_col[i] = 8 * (u % units);
    }
    const int x_tok = tid >> 3, x_col = 8 * (tid & 7);
    const bool x_in = slab * kSlab + x_col < a.vdim;
    const __bf16* rows = a.xbc + (row0 - a.xbc_row0) * a.xbc_stride;
    const __bf16* b_src = rows + inner + grp * N;
    const __bf16* c_src = b_src + a.groups * N;
    const __bf16* x_src = rows + h * a.vdim + (x_in ? slab * kSlab + x_col : 0);
    const __bf16* dt_src = a.proj + (int64_t)row0 * a.proj_stride + a.dt_off + h;
    u32x4_t breg[NU], creg[NU], xreg;
    __bf16 dtreg;
    auto fetch = [&](int c) {                                    // chunk c; tokens behind the last one re-read it
        const int last = count - 1, t0 = c * kC;
        auto tok = [&](int i) { return t0 + i < last ? t0 + i : last; };
#pragma unroll
        for (int i = 0; i < NU; ++i) {
            const int64_t r = tok(u_tok[i] > 0 ? u_tok[i] : 0) * a.xbc_stride;
            breg[i] = *reinterpret_cast<const u32x4_t*>(b_src + r + u_col[i]);
            if constexpr (OUT) creg[i] = *reinterpret_cast<const u32x4_t*>(c_src + r + u_col[i]);
        }
        xreg = *reinterpret_cast<const u32x4_t*>(x_src + tok(x_tok) * a.xbc_stride);
    };
    auto fetch_dt = [&](int c) {
        const int t = c * kC + (lane & 31);
        dtreg = dt_src[(int64_t)(t < count ? t : count - 1) * a.proj_stride];
    };
    const float a2 = -expf(a.a_log[h]) * kLog2e, bias = a.dt_bias[h], dh = a.d[h];
    float total = 0.f;                                           // log2 of the segment's decay
    fetch(0);
    fetch_dt(wave);
    for (int c = 0; c < chunks; ++c) {
        __syncthreads();
        if (c % kAhead == 0) {                                   // this wavefront's chunk is c + wave
            const float dt = (c + wave) * kC + (lane & 31) < count ? softplus_f((float)dtreg + bias) : 0.f;
            float G = fmaxf(a2 * dt, -160.f);                    // nothing is left beyond, and sums stay precise
#pragma unroll
            for (int m = 1; m < kC; m <<= 1) {
                const float up = __shfl_up(G, m, 32);
                G += (lane & 31) >= m ? up : 0.f;
            }
            const float end = __shfl(G, kC - 1, 64);
            if (lane < kC) {
                sums[wave][lane] = G;
                steps[wave][lane] = dt;
                weights[wave][lane] = __builtin_amdgcn_exp2f(end - G) * dt;
            }
            fetch_dt(c + kAhead + wave);
        }
#pragma unroll
        for (int i = 0; i < NU; ++i)
            if (u_tok[i] >= 0) {
                *reinterpret_cast<u32x4_t*>(bbuf + u_tok[i] * kRow + 2 * u_col[i]) = breg[i];
                if constexpr (OUT) *reinterpret_cast<u32x4_t*>(cbuf + u_tok[i] * kRow + 2 * u_col[i]) = creg[i];
            }
        if (x_in) *reinterpret_cast<u32x4_t*>(xbuf + x_tok * kXRow + 2 * x_col) = xreg;
        if (c + 1 < chunks) fetch(c + 1);
        __syncthreads();
        const float* sum = sums[c % kAhead];
        const float* step = steps[c % kAhead];
        const float* weight = weights[c % kAhead];
        const float G_end = sum[kC - 1];
        // x of this wavefront's columns: lane (g, n) has tokens 8 g .. 8 g + 7 of column n
        const unsigned char* xr = xbuf + (8 * g + (n >> 2)) * kXRow + (n & 3) * 8 + 32 * wave;
        const i16x4 xlo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)xr);
        const i16x4 xhi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(xr + 4 * kXRow));
        const bf16x8_t xf = __builtin_bit_cast(bf16x8_t, (i16x8)__builtin_shufflevector(xlo, xhi, 0, 1, 2, 3, 4, 5, 6, 7));
        f32x4_t y[2];
        if constexpr (OUT) {
            // products C_i B_j of one 16 x 16 tile: lane (g, n) gets tokens j = 4 g + e and i = n of it
            const int sj = wave >> 1, ti = wave & 1;
            f32x4_t m = {0.f, 0.f, 0.f, 0.f};
            if (sj <= ti) {
#pragma unroll
                for (int k = 0; k < NS; ++k) {
                    const bf16x8_t bf = *reinterpret_cast<const bf16x8_t*>(bbuf + (16 * sj + n) * kRow + 64 * k + 16 * g);
                    const bf16x8_t cf = *reinterpret_cast<const bf16x8_t*>(cbuf + (16 * ti + n) * kRow + 64 * k + 16 * g);
                    m = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf, cf, m, 0, 0, 0);
                }
            }
            const int i = 16 * ti + n, j0 = 16 * sj + 4 * g;
            float v[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int j = j0 + e;
                v[e] = j <= i ? m[e] * __builtin_amdgcn_exp2f(sum[i] - sum[j]) * step[j] : 0.f;
                if (j == i) v[e] += dh;
            }
            uint32_t p[2][2];
            split<2, 4>(v, p);
#pragma unroll
            for (int k = 0; k < 2; ++k)
                *reinterpret_cast<uint2*>(mbuf + k * kC * kMRow + i * kMRow + 2 * j0) = uint2{p[k][0], p[k][1]};
            // products of the state: lane (g, n) gets columns 4 g + e for token n
            y[0] = y[1] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < NS; ++k) {
                float sv[8];
#pragma unroll
                for (int e = 0; e < 8; ++e) sv[e] = s[2 * k + e / 4][e % 4];
                bf16x8_t sp[2];
                split_frags<2>(sv, sp);
#pragma unroll
                for (int t = 0; t < 2; ++t) {
                    const unsigned char* cr = cbuf + (16 * t + n) * kRow + 64 * k + 8 * g;
                    const uint2 lo = *reinterpret_cast<const uint2*>(cr), hi = *reinterpret_cast<const uint2*>(cr + 32);
                    const bf16x8_t cf = __builtin_bit_cast(bf16x8_t, u32x4_t{lo.x, lo.y, hi.x, hi.y});
                    y[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sp[1], cf, y[t], 0, 0, 0);
                    y[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sp[0], cf, y[t], 0, 0, 0);
                }
            }
#pragma unroll
            for (int t = 0; t < 2; ++t) y[t] *= __builtin_amdgcn_exp2f(sum[16 * t + n]);
        }
        // the state
        float wx[8], xv[8];
        widen(__builtin_bit_cast(u32x4_t, xf), xv);
#pragma unroll
        for (int e = 0; e < 8; ++e) wx[e] = xv[e] * weight[8 * g + e];
        bf16x8_t xp[3];
        split_frags<3>(wx, xp);
        const float carry = __builtin_amdgcn_exp2f(G_end);
        total += G_end;
#pragma unroll
        for (int t = 0; t < 2 * NS; ++t) {
            const unsigned char* br = bbuf + (8 * g + (n >> 2)) * kRow + (n & 3) * 8 + 32 * t;
            const i16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)br);
            const i16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(br + 4 * kRow));
            const bf16x8_t bf = __builtin_bit_cast(bf16x8_t, (i16x8)__builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
            s[t] *= carry;
#pragma unroll
            for (int k = 2; k >= 0; --k) s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf, xp[k], s[t], 0, 0, 0);
        }
        if constexpr (OUT) {
            __syncthreads();
#pragma unroll
            for (int t = 0; t < 2; ++t) {
#pragma unroll
                for (int k = 1; k >= 0; --k) {
                    const bf16x8_t mf = *reinterpret_cast<const bf16x8_t*>(mbuf + k * kC * kMRow + (16 * t + n) * kMRow + 16 * g);
                    y[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xf, mf, y[t], 0, 0, 0);
                }
                const int tok = c * kC + 16 * t + n;
                if (tok < count && v0 + 4 * g < a.vdim) {
                    bf16x4_t o;
#pragma unroll
                    for (int e = 0; e < 4; ++e) o[e] = (__bf16)y[t][e];
                    *reinterpret_cast<bf16x4_t*>(a.y + (row0 + tok) * a.y_stride + h * a.vdim + v0 + 4 * g) = o;
                }
            }
        }
    }
    if (!OUT && slab == 0 && tid == 0) args.ws_decay[rec] = total;
    if (OUT && !last_seg) return;
    if (col_live)
#pragma unroll
        for (int t = 0; t < 2 * NS; ++t)
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (16 * t + 4 * g + e < N) to[(int64_t)(16 * t + 4 * g + e) * a.vdim + v0 + n] = s[t][e];
}

// final states of segments from zero -> the states in front of the segments
__global__ void __launch_bounds__(kThreads) ssm_join_kernel(ChunkArgs args) {
    const SsmArgs<__bf16>& a = args.a;
    const Span span = args.spans[blockIdx.z];
    const int h = blockIdx.y;
    const int64_t state_len = (int64_t)a.state_n * a.vdim, i = (int64_t)blockIdx.x * kThreads + threadIdx.x;
    if (i >= state_len || span.slot < 0 || span.slot >= a.num_slots) return;
    float cur = span.pos0 > 0 ? a.state[((int64_t)span.slot * a.heads + h) * state_len + i] : 0.f;
    const int segs = (span.count + args.seg_len - 1) / args.seg_len;
    for (int k = 0; k < segs; ++k) {
        const int64_t rec = ((int64_t)blockIdx.z * args.max_seg + k) * a.heads + h;
        float* w = args.ws + rec * state_len + i;
        const float own = k + 1 < segs ? *w : 0.f, decay = k + 1 < segs ? __builtin_amdgcn_exp2f(args.ws_decay[rec]) : 0.f;
        *w = cur;
        cur = cur * decay + own;
    }
}

// ------------------------------------------------------------------ gate and norm
template <class T>
struct NormArgs {
    SsmArgs<T> a;
    const float* norm;                     // [heads * vdim]
    int parts; float eps;
    const int32_t* ring_slot;              // [row][2]: slot, rows of the portion that follow
    const int64_t* positions;
    int64_t portion_row;                   // rows from here on belong to portions
    T* out; int64_t out_stride;
};

template <class T, int VEC>
__global__ void __launch_bounds__(kThreads) ssm_norm_kernel(NormArgs<T> b) {
    __shared__ float part[kThreads / 64];
    const SsmArgs<T>& a = b.a;
    const int64_t row = blockIdx.x;
    const int size = a.heads * a.vdim / b.parts, c0 = blockIdx.y * size, tid = threadIdx.x;
    const T* y = a.y + row * a.y_stride + c0;
    const T* z = a.proj + row * a.proj_stride + a.z_off + c0;
    constexpr int kKeep = 4;               // chunks kept between the sum and the result; more are computed twice
    float x[kKeep][VEC], ss = 0.f;
    auto gated = [&](int c, float (&v)[VEC]) {
        float w[VEC];
        load_elems<VEC>(y + c, v);
        load_elems<VEC>(z + c, w);
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] *= silu_f(w[e]);
    };
#pragma unroll
    for (int j = 0; j < kKeep; ++j) {
        const int c = (tid + j * kThreads) * VEC;
        if (c < size) {
            gated(c, x[j]);
#pragma unroll
            for (int e = 0; e < VEC; ++e) ss += x[j][e] * x[j][e];
        }
    }
    for (int c = (tid + kKeep * kThreads) * VEC; c < size; c += kThreads * VEC) {
        float v[VEC];
        gated(c, v);
#pragma unroll
        for (int e = 0; e < VEC; ++e) ss += v[e] * v[e];
    }
    const float rs = rsqrtf(block_sum<kThreads / 64>(ss, part) / (float)size + b.eps);
    auto put = [&](int c, float (&v)[VEC]) {
        float w[VEC];
        load_elems<VEC>(b.norm + c0 + c, w);
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] *= rs * w[e];
        store_elems<VEC>(b.out + row * b.out_stride + c0 + c, v);
    };
#pragma unroll
    for (int j = 0; j < kKeep; ++j) {
        const int c = (tid + j * kThreads) * VEC;
        if (c < size) put(c, x[j]);
    }
    for (int c = (tid + kKeep * kThreads) * VEC; c < size; c += kThreads * VEC) {
        float v[VEC];
        gated(c, v);
        put(c, v);
    }
    if (row >= b.portion_row && blockIdx.y == 0 && b.ring_slot[2 * row + 1] < a.taps - 1) {
        const int slot = b.ring_slot[2 * row];
        if (slot < 0 || slot >= a.num_slots) return;
        T* ring = a.ring + ((int64_t)slot * a.taps + b.positions[row] % a.taps) * a.channels;
        const T* in = a.proj + row * a.proj_stride + a.x_off;
        for (int c = tid; c < a.channels; c += kThreads) ring[c] = in[c];
    }
}

// ------------------------------------------------------------------ launches
bool chunked(int elem, int64_t vdim, int64_t state_n) { return elem == INFER_ELEM_BF16 && vdim % 8 == 0 && state_n % 8 == 0 && state_n <= 256; }

// segments that portions are cut into, so that enough workgroups run: tokens per segment and their largest number
void segments(int64_t heads, int64_t slabs, int64_t num_spans, int64_t max_span, int64_t& seg_len, int64_t& max_seg) {
    const int64_t units = heads * slabs * num_spans, chunks = (max_span + kC - 1) / kC;
    int64_t want = units > 0 && units < 512 ? (768 + units - 1) / units : 1;       // three workgroups per compute unit
    if (want > chunks / 4) want = chunks / 4;              // no segment shorter than four chunks
    if (want < 1) want = 1;
    const int64_t per = (chunks + want - 1) / want;
    seg_len = (per > 0 ? per : 1) * kC;
    max_seg = max_span > 0 ? (max_span + seg_len - 1) / seg_len : 1;
}

template <int NS>
int launch_chunks(const ChunkArgs& c, int64_t num_spans, hipStream_t st) {
    const dim3 grid((unsigned)(c.slabs * c.max_seg), (unsigned)c.a.heads, (unsigned)num_spans), block(kThreads);
    if (c.max_seg > 1) {
        hipLaunchKernelGGL((ssm_chunk_kernel<NS, false>), grid, block, 0, st, c);
        const int64_t state_len = (int64_t)c.a.state_n * c.a.vdim;
        hipLaunchKernelGGL(ssm_join_kernel, dim3((unsigned)((state_len + kThreads - 1) / kThreads), (unsigned)c.a.heads, (unsigned)num_spans),
                           block, 0, st, c);
    }
    hipLaunchKernelGGL((ssm_chunk_kernel<NS, true>), grid, block, 0, st, c);
    return (int)hipGetLastError();
}

template <class T>
int portions(SsmArgs<T>& a, const Span* spans, int64_t num_spans, int64_t max_span, int64_t row0, int64_t n, T* xbc, float* ws,
             int64_t ws_floats, hipStream_t st) {
    const int64_t rows = n - row0;
    if (!spans || !xbc || num_spans < 1 || num_spans > 65535 || max_span < 1 || max_span > rows) return INFER_KV_EINVAL;
    a.xbc = xbc;
    a.xbc_stride = a.channels;
    a.xbc_row0 = row0;
    const bool vec = a.channels % 8 == 0 && a.proj_stride % 8 == 0 && a.x_off % 8 == 0 && ptr_aligned(a.proj, 16) && ptr_aligned(xbc, 16) &&
                     ptr_aligned(a.ring, 16) && ptr_aligned(a.conv_bias, 16);
    const int64_t units = vec ? a.channels / 8 : a.channels, token_blocks = (max_span + kConvTokens - 1) / kConvTokens;
    if (token_blocks > 65535) return INFER_KV_EINVAL;
    const dim3 grid((unsigned)((units + kThreads - 1) / kThreads), (unsigned)token_blocks, (unsigned)num_spans), block(kThreads);
    if (vec && a.taps == 4) hipLaunchKernelGGL((ssm_conv_kernel<T, 8, 4>), grid, block, 0, st, a, spans, xbc);
    else if (vec) hipLaunchKernelGGL((ssm_conv_kernel<T, 8, 0>), grid, block, 0, st, a, spans, xbc);
    else hipLaunchKernelGGL((ssm_conv_kernel<T, 1, 0>), grid, block, 0, st, a, spans, xbc);
    if constexpr (sizeof(T) == 2) {
        if (chunked(INFER_ELEM_BF16, a.vdim, a.state_n) && vec && a.y_stride % 4 == 0 && ptr_aligned(a.y, 8)) {
            ChunkArgs c{a, spans, 0, 0, (a.vdim + kSlab - 1) / kSlab, nullptr, nullptr};
            int64_t seg_len, max_seg;
            segments(a.heads, c.slabs, num_spans, max_span, seg_len, max_seg);
            c.seg_len = (int)seg_len;
            c.max_seg = (int)max_seg;
            if (max_seg > 1) {
                const int64_t records = num_spans * max_seg * a.heads, len = (int64_t)a.state_n * a.vdim;
                if (!ws || ws_floats < records * (len + 1)) return INFER_KV_EWORKSPACE;
                c.ws = ws;
                c.ws_decay = ws + records * len;
            }
            if (a.state_n <= 64) return launch_chunks<2>(c, num_spans, st);
            if (a.state_n <= 128) return launch_chunks<4>(c, num_spans, st);
            return launch_chunks<8>(c, num_spans, st);
        }
    }
    const dim3 sgrid((unsigned)((a.vdim + 15) / 16), (unsigned)a.heads, (unsigned)num_spans);
    if (a.state_n <= 64) hipLaunchKernelGGL((ssm_scan_any_kernel<T, 4>), sgrid, block, 0, st, a, spans);
    else if (a.state_n <= 256) hipLaunchKernelGGL((ssm_scan_any_kernel<T, 16>), sgrid, block, 0, st, a, spans);
    else if (a.state_n <= 1024) hipLaunchKernelGGL((ssm_scan_any_kernel<T, 64>), sgrid, block, 0, st, a, spans);
    else return INFER_KV_EUNSUPPORTED;
    return (int)hipGetLastError();
}

bool size_in(int64_t v, int64_t lo, int64_t hi) { return v >= lo && v <= hi; }

}  // namespace

extern "C" int64_t infer_state_space_workspace_floats(int elem, int64_t heads, int64_t vdim, int64_t state_n, int64_t num_spans,
                                                      int64_t max_span) {
    if (!chunked(elem, vdim, state_n) || heads < 1 || num_spans < 1 || max_span < 1) return 0;
    int64_t seg_len, max_seg;
    segments(heads, (vdim + kSlab - 1) / kSlab, num_spans, max_span, seg_len, max_seg);
    return max_seg > 1 ? num_spans * max_seg * heads * (state_n * vdim + 1) : 0;
}

extern "C" int infer_state_space(int elem, const void* proj, int64_t proj_stride, int64_t z_off, int64_t x_off, int64_t dt_off,
                                 int64_t heads, int64_t vdim, int64_t state_n, int64_t groups, int64_t taps, const float* conv,
                                 const float* conv_bias, const float* dt_bias, const float* a_log, const float* d, const float* norm,
                                 int64_t norm_parts, float eps, void* ring, float* state, int64_t num_slots, const int32_t* slots,
                                 const int64_t* positions, int64_t decode_rows, const int32_t* spans, int64_t num_spans,
                                 int64_t max_span, const int32_t* ring_slot, int64_t n, void* xbc, void* y, float* workspace,
                                 int64_t workspace_floats, void* out, int64_t out_stride, void* stream) {
    if (n < 0 || n > 0x7fffffff || decode_rows < 0 || decode_rows > n) return INFER_KV_EINVAL;
    if (n == 0) return INFER_KV_OK;
    if (!size_in(heads, 1, 4096) || !size_in(vdim, 1, 1024) || !size_in(state_n, 1, 1024) || !size_in(groups, 1, heads) || heads % groups ||
        !size_in(taps, 1, 64) || norm_parts < 1 || heads * vdim % norm_parts || norm_parts > 65535 || num_slots < 1)
        return INFER_KV_EINVAL;
    const int64_t inner = heads * vdim, channels = inner + 2 * groups * state_n;
    if (!proj || !conv || !conv_bias || !dt_bias || !a_log || !d || !norm || !ring || !state || !y || !out || !positions || z_off < 0 ||
        x_off < 0 || dt_off < 0 || z_off + inner > proj_stride || x_off + channels > proj_stride || dt_off + heads > proj_stride ||
        out_stride < inner || proj_stride > (1 << 24) || (decode_rows > 0 && !slots) || (decode_rows < n && !ring_slot))
        return INFER_KV_EINVAL;
    hipStream_t st = (hipStream_t)stream;
    auto go = [&](auto zero) -> int {
        using T = decltype(zero);
        SsmArgs<T> a{(const T*)proj, proj_stride, (int)z_off, (int)x_off, (int)dt_off, (int)heads, (int)vdim, (int)state_n, (int)groups,
                     (int)channels, (int)taps, conv, conv_bias, dt_bias, a_log, d, (T*)ring, state, (int)num_slots, (T*)y, inner, nullptr, 0, 0};
        if (decode_rows > 0) {
            if (decode_rows > 65535) return INFER_KV_EINVAL;
            const bool vec = vdim % 4 == 0 && ptr_aligned(state, 16);
            const int64_t quads = vdim / (vec ? 4 : 1);
            if (quads > kThreads) return INFER_KV_EUNSUPPORTED;
            const size_t lds = sizeof(float) * ((vdim + 3) / 4 * 4 + 2 * ((state_n + 3) / 4 * 4) + kThreads / quads * vdim);
            const dim3 grid((unsigned)heads, (unsigned)decode_rows), block(kThreads);
            if (vec) hipLaunchKernelGGL((ssm_step_kernel<T, 4>), grid, block, lds, st, a, slots, positions);
            else hipLaunchKernelGGL((ssm_step_kernel<T, 1>), grid, block, lds, st, a, slots, positions);
        }
        if (decode_rows < n) {
            const int rc = portions<T>(a, (const Span*)spans, num_spans, max_span, decode_rows, n, (T*)xbc, workspace, workspace_floats, st);
            if (rc) return rc;
        }
        const NormArgs<T> b{a, norm, (int)norm_parts, eps, ring_slot, positions, decode_rows, (T*)out, out_stride};
        const int64_t size = inner / norm_parts;
        const bool vec = size % 8 == 0 && inner % 8 == 0 && proj_stride % 8 == 0 && z_off % 8 == 0 && out_stride % 8 == 0 &&
                         ptr_aligned(proj, 16) && ptr_aligned(y, 16) && ptr_aligned(out, 16) && ptr_aligned(norm, 16);
        const dim3 grid((unsigned)n, (unsigned)norm_parts), block(kThreads);
        if (vec) hipLaunchKernelGGL((ssm_norm_kernel<T, 8>), grid, block, 0, st, b);
        else hipLaunchKernelGGL((ssm_norm_kernel<T, 1>), grid, block, 0, st, b);
        return (int)hipGetLastError();
    };
    if (elem == INFER_ELEM_BF16) return go(__bf16(0.f));
    if (elem == INFER_ELEM_F32) return go(0.f);
    return INFER_KV_EUNSUPPORTED;
}
