// Linear attention with a constant decay per head, for gfx950 (MI355X).  Per head, over a float32 state S[dim][vdim]:
//     S <- d S + k v^T ;   o = c S^T q
// (d and c constants), q, k and v being projections, optionally behind silu (q, k, v) or a rotary embedding (q, k;
// entry i turns with entry i + pairs).  Behind it an RMS norm over each head or over all heads at once and an output gate.
//
//   decay_step_kernel     one token per sequence (decode): one workgroup per (sequence, head), the state passes
//                         through registers once; with a norm per head the norm and the gate are in it too
//   decay_chunk_kernel    prompt portions in chunks of 32 tokens on bf16 matrix instructions
//   decay_join_kernel     carries the state over the segments that a long portion is cut into
//   decay_scan_any_kernel prompt portions of any size and element type, token by token
//   decay_out_kernel      norm and gate of whole rows
//
// A sequence at position 0 starts from a zero state whatever its slot holds, so a slot needs no clearing when another
// sequence takes it over.  d is held as a sum of two floats: its rounding error would enter a long memory once per
// token.
//
// Chunk form.  With S the state before a chunk of n tokens,
//     o_i = c (d^{i+1} q_i^T S + sum_{j<=i} d^{i-j} (q_i k_j) v_j) ,   S' = d^n S + sum_j k_j (d^{n-1-j} v_j)^T .
// What enters the state is held to float precision although the products run as bf16: a float is the exact sum of
// three bf16 numbers of 8 bits each, and the products of the pieces are added up in float32, without those below 2^-24
// of the result.  The products of the output, which leave the recurrence and are rounded to bf16 behind it, take two
// pieces (2^-17).  Projections, with silu behind them or not, are bf16 already: one piece.
// A portion with few heads is cut into segments that run side by side: first every segment from a zero state, keeping
// only its final state, then the states are joined in order, then every segment with its outputs.
#include <type_traits>

#include "elem.h"
#include "pieces.h"

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

// ------------------------------------------------------------------ chunks of 32 tokens
typedef short i16x4 __attribute__((ext_vector_type(4)));
typedef short i16x8 __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) i16x4 lds_i16x4;
typedef uint32_t u32x2_t __attribute__((ext_vector_type(2)));

constexpr int kC = 32;                           // tokens per chunk

struct ChunkArgs {
    DecayArgs<__bf16> a;
    DecayOutArgs<__bf16> b;
    bool finish;                                 // norm (per head) and gate here; a.o is not written
    const Span* spans;
    int seg_len, max_seg, slabs;                 // tokens per segment (a multiple of kC), segments of the longest span
    float* ws;                                   // [span][max_seg][heads][dim_pad][vdim_pad], if max_seg > 1
};

// sum of the products of pieces i of x and j of y with i + j < MOST, the small ones first
template <int MOST, int PX, int PY>
__device__ __forceinline__ f32x4_t mfma_pieces(const bf16x8_t (&x)[PX], const bf16x8_t (&y)[PY], f32x4_t acc) {
#pragma unroll
    for (int k = MOST - 1; k >= 0; --k)
#pragma unroll
        for (int i = 0; i <= k; ++i)
            if (i < PX && k - i < PY) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x[i], y[k - i], acc, 0, 0, 0);
    return acc;
}

__device__ __forceinline__ u32x4_t silu8(u32x4_t x) {
    float y[8];
    widen(x, y);
    bf16x8_t r;
#pragma unroll
    for (int i = 0; i < 8; ++i) r[i] = (__bf16)silu_f(y[i]);
    return __builtin_bit_cast(u32x4_t, r);
}

// A workgroup of four wavefronts serves one head and 64 VT columns of its state over the chunks of one segment.
// Wavefront w owns the columns 16 VT w .. and their part of the state, DT tiles of 32 rows, as accumulators: lane (g, n)
// holds rows 16 t + 4 g + e of column n.  That is an operand of the next product as it lies, when the rows of a
// k-step of 32 are taken in the order 16 tau + 4 g + e.  The 32 x 32 products q_i k_j are shared out over the
// wavefronts, weighted, and exchanged through LDS while the products with the state run.
// PC: pieces of k (3 behind a rotation, otherwise 1; q then has 2).  OUT = false: only the final state, from zero.
template <int DT, int VT, int PC, bool OUT>
__global__ void __launch_bounds__(256, 2) decay_chunk_kernel(ChunkArgs args) {
    constexpr int kRow = DT * 64 + 16, kMat = kC * kRow;         // bytes: a token of q or k, one piece of a chunk
    constexpr int kSlab = 64 * VT;
    constexpr int PQ = PC == 3 ? 2 : 1;                          // pieces of q
    constexpr int kVRow = 2 * kSlab + 16, kPRow = 2 * kC + 16, kPMat = kC * kPRow;
    constexpr int NU = DT > 4 ? DT / 4 : 1;                      // units of 16 columns of q and k per thread
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];
    const DecayArgs<__bf16>& a = args.a;
    unsigned char* kbuf = lds;                                   // [PC][kMat]
    unsigned char* vbuf = kbuf + PC * kMat;                      // [kC][kVRow]
    unsigned char* qbuf = vbuf + kC * kVRow;                     // [PQ][kMat]
    unsigned char* pbuf = qbuf + PQ * kMat;                      // [2][kPMat]
    float* squares = reinterpret_cast<float*>(pbuf + 2 * kPMat); // [4][kC]
    const int tid = threadIdx.x, lane = tid & 63, g = lane >> 4, n = lane & 15;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int h = blockIdx.y, slab = blockIdx.x % args.slabs, seg = blockIdx.x / args.slabs;
    const Span span = args.spans[blockIdx.z];
    const int first = seg * args.seg_len;
    if (span.slot < 0 || span.slot >= a.num_slots || first >= span.count) return;
    const bool last_seg = first + args.seg_len >= span.count;
    if (!OUT && last_seg) return;                                // nobody needs its final state yet
    const int count = last_seg ? span.count - first : args.seg_len;
    const int row0 = span.row0 + first, pos0 = span.pos0 + first, chunks = (count + kC - 1) / kC;
    const int v0 = slab * kSlab + wave * 16 * VT;                // this wavefront's first column
    const bool live = v0 < a.vdim_pad;
    const float log2d = a.decay[2 * a.heads + h];
    const int64_t state_len = (int64_t)a.dim_pad * a.vdim_pad;
    float* from = a.state + ((int64_t)span.slot * a.heads + h) * state_len;
    float* to = from;
    if (args.max_seg > 1) {
        float* ws = args.ws + (((int64_t)blockIdx.z * args.max_seg + seg) * a.heads + h) * state_len;
        if (OUT) from = ws;
        else to = ws;
    }
    const bool load = OUT && (args.max_seg > 1 || span.pos0 > 0);

    f32x4_t s[2 * DT][VT];
#pragma unroll
    for (int t = 0; t < 2 * DT; ++t)
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            s[t][v] = f32x4_t{0.f, 0.f, 0.f, 0.f};
            const int col = v0 + 16 * v + n;
            if (load && col < a.vdim_pad)
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (16 * t + 4 * g + e < a.dim_pad) s[t][v][e] = from[(int64_t)(16 * t + 4 * g + e) * a.vdim_pad + col];
        }

    // entries behind the real sizes stay zero
    for (int i = tid; i < ((PC + (OUT ? PQ : 0)) * kMat + kC * kVRow) / 16; i += 256) reinterpret_cast<u32x4_t*>(lds)[i] = u32x4_t{0u, 0u, 0u, 0u};

    // unit i of this thread: token, and two blocks of 8 columns, which turn together if they are rotated
    // (token -1: there is no such unit; its loads repeat another one and are not stored)
    const int half = PC == 3 ? a.rot_pairs : a.dim / 2, units = a.dim / 16;
    int u_tok[NU], u_b0[NU], u_b1[NU], u_pair[NU];
    const __bf16* u_src[NU];
    const float* u_cs[NU];
#pragma unroll
    for (int i = 0; i < NU; ++i) {
        const int u = tid + 256 * i, w = u % units, rotated = half / 8;
        u_tok[i] = u < kC * units ? u / units : -1;
        u_pair[i] = PC == 3 && w < rotated ? 8 * w : -1;
        u_b0[i] = w < rotated ? 8 * w : 2 * half + 16 * (w - rotated);
        u_b1[i] = w < rotated ? 8 * w + half : u_b0[i] + 8;
        u_src[i] = a.proj + (int64_t)(row0 + (u_tok[i] > 0 ? u_tok[i] : 0)) * a.proj_stride + h * a.dim;
        u_cs[i] = a.table + 2 * (u_pair[i] > 0 ? u_pair[i] : 0);
    }
    int v_tok[VT], v_col[VT];
    const __bf16* v_src[VT];
#pragma unroll
    for (int i = 0; i < VT; ++i) {
        const int x = tid + 256 * i;
        v_tok[i] = x / (kSlab / 8);
        v_col[i] = slab * kSlab + 8 * (x % (kSlab / 8));
        v_src[i] = a.proj + (int64_t)(row0 + v_tok[i]) * a.proj_stride + a.v_off + h * a.vdim + (v_col[i] < a.vdim ? v_col[i] : 0);
    }
    const int64_t step = kC * a.proj_stride;
    u32x4_t kreg[NU][2], qreg[NU][2], vreg[VT];
    f32x4_t creg[PC == 3 ? NU : 1][4];
    // requests chunk c, the one behind the last request; no branches, so that nothing waits for a request before its use
    auto fetch = [&](int c) {
        const int last = count - c * kC - 1;                     // tokens behind the last one re-read it
#pragma unroll
        for (int i = 0; i < NU; ++i) {
            const int tok = u_tok[i] > 0 ? u_tok[i] : 0, over = tok > last ? tok - last : 0;
            const __bf16* r = u_src[i] - over * a.proj_stride;
            kreg[i][0] = *reinterpret_cast<const u32x4_t*>(r + a.k_off + u_b0[i]);
            kreg[i][1] = *reinterpret_cast<const u32x4_t*>(r + a.k_off + u_b1[i]);
            if constexpr (OUT) {
                qreg[i][0] = *reinterpret_cast<const u32x4_t*>(r + a.q_off + u_b0[i]);
                qreg[i][1] = *reinterpret_cast<const u32x4_t*>(r + a.q_off + u_b1[i]);
            }
            u_src[i] += step;
            if constexpr (PC == 3) {
                int64_t pos = pos0 + c * kC + tok;
                pos = pos < 0 ? 0 : (pos >= a.max_pos ? a.max_pos - 1 : pos);
                const float* cs = u_cs[i] + pos * (2 * a.rot_pairs);
#pragma unroll
                for (int e = 0; e < 4; ++e) creg[i][e] = *reinterpret_cast<const f32x4_t*>(cs + 4 * e);
            }
        }
#pragma unroll
        for (int i = 0; i < VT; ++i) {
            const int over = v_tok[i] > last ? v_tok[i] - last : 0;
            vreg[i] = *reinterpret_cast<const u32x4_t*>(v_src[i] - over * a.proj_stride);
            v_src[i] += step;
        }
    };
    // the two blocks of a unit to LDS, in PB pieces
    auto put_unit = [&](auto pieces, unsigned char* r, int i, const u32x4_t (&x)[2], bool in) {
        constexpr int PB = decltype(pieces)::value;
        if constexpr (PB == 1) {
            u32x4_t y0 = x[0], y1 = x[1];
            if (a.silu) { y0 = silu8(y0); y1 = silu8(y1); }
            if (!in) y0 = y1 = u32x4_t{0u, 0u, 0u, 0u};
            *reinterpret_cast<u32x4_t*>(r + 2 * u_b0[i]) = y0;
            *reinterpret_cast<u32x4_t*>(r + 2 * u_b1[i]) = y1;
        } else {
            float y0[8], y1[8];
            widen(x[0], y0);
            widen(x[1], y1);
            if (u_pair[i] >= 0)
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    const float cv = creg[i][e / 2][2 * (e & 1)], sv = creg[i][e / 2][2 * (e & 1) + 1], u = y0[e];
                    y0[e] = u * cv - y1[e] * sv;
                    y1[e] = y1[e] * cv + u * sv;
                }
            if (!in)
#pragma unroll
                for (int e = 0; e < 8; ++e) y0[e] = y1[e] = 0.f;
            bf16x8_t f[PB];
            split_frags<PB>(y0, f);
#pragma unroll
            for (int k = 0; k < PB; ++k) *reinterpret_cast<bf16x8_t*>(r + k * kMat + 2 * u_b0[i]) = f[k];
            split_frags<PB>(y1, f);
#pragma unroll
            for (int k = 0; k < PB; ++k) *reinterpret_cast<bf16x8_t*>(r + k * kMat + 2 * u_b1[i]) = f[k];
        }
    };
    auto put = [&](int c) {
        const int left = count - c * kC;
#pragma unroll
        for (int i = 0; i < NU; ++i) {
            if (u_tok[i] < 0) continue;
            put_unit(std::integral_constant<int, PC>{}, kbuf + u_tok[i] * kRow, i, kreg[i], u_tok[i] < left);
            if constexpr (OUT) put_unit(std::integral_constant<int, PQ>{}, qbuf + u_tok[i] * kRow, i, qreg[i], u_tok[i] < left);
        }
#pragma unroll
        for (int i = 0; i < VT; ++i) {
            if (v_col[i] >= a.vdim) continue;
            u32x4_t y = a.silu ? silu8(vreg[i]) : vreg[i];
            if (v_tok[i] >= left) y = u32x4_t{0u, 0u, 0u, 0u};
            *reinterpret_cast<u32x4_t*>(vbuf + v_tok[i] * kVRow + 2 * (v_col[i] - slab * kSlab)) = y;
        }
    };

    // weights of the products: this lane's query column n of tile w / 2, keys 4 g + e of tile w % 2
    float pw[4], qw[2], vw[8];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const int dist = 16 * (wave >> 1) + n - (16 * (wave & 1) + 4 * g + e);
        pw[e] = dist >= 0 ? a.scale * exp2f(dist * log2d) : 0.f;
    }
#pragma unroll
    for (int t = 0; t < 2; ++t) qw[t] = a.scale * exp2f((16 * t + n + 1) * log2d);
    auto value_weights = [&](int tokens) {
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const int after = tokens - 1 - (8 * g + i);
            vw[i] = exp2f((after > 0 ? after : 0) * log2d);      // values behind the last token are zero
        }
    };
    value_weights(kC);
    float chunk_decay = exp2f(kC * log2d);

#pragma unroll
    for (int t = 0; t < 2 * DT; ++t)
#pragma unroll
        for (int v = 0; v < VT; ++v)
#pragma unroll
            for (int e = 0; e < 4; ++e) {                        // the state has arrived: nothing in the loop waits for it
                float x = s[t][v][e];
                asm volatile("" : "+v"(x));
                s[t][v][e] = x;
            }
    fetch(0);
    __syncthreads();                                             // the zero fill
    for (int c = 0; c < chunks; ++c) {
        put(c);
        __syncthreads();
        const int left = count - c * kC;
        fetch(c + 1);
        if (left < kC) {
            value_weights(left);
            chunk_decay = exp2f(left * log2d);
        }
        u32x2_t gate[VT][2];                                     // of this chunk's results, for when they are there
        f32x4_t acc[VT][2];                                      // rows are columns of the state, columns queries
        if constexpr (OUT) {
            // ---- d^(i-j) q_i k_j: rows are keys, columns queries; the tile above the diagonal is all zeros
            {
                f32x4_t p = {0.f, 0.f, 0.f, 0.f};
                if (wave != 1) {
                    const unsigned char* kr = kbuf + (16 * (wave & 1) + n) * kRow + 16 * g;
                    const unsigned char* qr = qbuf + (16 * (wave >> 1) + n) * kRow + 16 * g;
#pragma unroll
                    for (int j = 0; j < DT; ++j) {
                        bf16x8_t kf[PQ], qf[PQ];
#pragma unroll
                        for (int k = 0; k < PQ; ++k) {
                            kf[k] = *reinterpret_cast<const bf16x8_t*>(kr + k * kMat + 64 * j);
                            qf[k] = *reinterpret_cast<const bf16x8_t*>(qr + k * kMat + 64 * j);
                        }
                        p = mfma_pieces<2>(kf, qf, p);
                    }
                }
                float x[4];
#pragma unroll
                for (int e = 0; e < 4; ++e) x[e] = p[e] * pw[e];
                uint32_t pp[2][2];
                split<2, 4>(x, pp);
                unsigned char* pr = pbuf + (16 * (wave >> 1) + n) * kPRow + 2 * (16 * (wave & 1) + 4 * g);
#pragma unroll
                for (int k = 0; k < 2; ++k) *reinterpret_cast<u32x2_t*>(pr + k * kPMat) = u32x2_t{pp[k][0], pp[k][1]};
            }
            // ---- q_i^T S
#pragma unroll
            for (int v = 0; v < VT; ++v)
#pragma unroll
                for (int t = 0; t < 2; ++t) acc[v][t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
            if (live)
#pragma unroll
                for (int j = 0; j < DT; ++j) {
                    bf16x8_t qf[2][PQ];
#pragma unroll
                    for (int t = 0; t < 2; ++t)
#pragma unroll
                        for (int k = 0; k < PQ; ++k) {
                            const unsigned char* qr = qbuf + k * kMat + (16 * t + n) * kRow + 64 * j + 8 * g;
                            const u32x2_t x = *reinterpret_cast<const u32x2_t*>(qr), y = *reinterpret_cast<const u32x2_t*>(qr + 32);
                            qf[t][k] = __builtin_bit_cast(bf16x8_t, u32x4_t{x[0], x[1], y[0], y[1]});
                        }
#pragma unroll
                    for (int v = 0; v < VT; ++v) {
                        float x[8];
#pragma unroll
                        for (int e = 0; e < 4; ++e) { x[e] = s[2 * j][v][e]; x[4 + e] = s[2 * j + 1][v][e]; }
                        bf16x8_t sf[2];
                        split_frags<2>(x, sf);
#pragma unroll
                        for (int t = 0; t < 2; ++t) acc[v][t] = mfma_pieces<2>(sf, qf[t], acc[v][t]);
                    }
                }
            if (args.finish)
#pragma unroll
                for (int v = 0; v < VT; ++v)
#pragma unroll
                    for (int t = 0; t < 2; ++t) {
                        const int tok = 16 * t + n < left ? 16 * t + n : left - 1, col = v0 + 16 * v + 4 * g;
                        gate[v][t] = *reinterpret_cast<const u32x2_t*>(args.b.gate + (int64_t)(row0 + c * kC + tok) * args.b.gate_stride +
                                                                       (int64_t)h * a.vdim + (col < a.vdim ? col : 0));
                    }
            __syncthreads();
        }
        if (live) {
            bf16x8_t vf[VT];                                     // values of tokens 8 g .. + 7, column n
            const unsigned char* vr = vbuf + (8 * g + (n >> 2)) * kVRow + (n & 3) * 8 + 32 * VT * wave;
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                const i16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(vr + 32 * v));
                const i16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(vr + 32 * v + 4 * kVRow));
                vf[v] = __builtin_bit_cast(bf16x8_t, (i16x8)__builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
            }
            if constexpr (OUT) {
                // ---- the chunk's own tokens
#pragma unroll
                for (int t = 0; t < 2; ++t) {
                    bf16x8_t pf[2];
#pragma unroll
                    for (int k = 0; k < 2; ++k) pf[k] = *reinterpret_cast<const bf16x8_t*>(pbuf + k * kPMat + (16 * t + n) * kPRow + 16 * g);
                    float ss = 0.f;
#pragma unroll
                    for (int v = 0; v < VT; ++v) {
                        acc[v][t] *= qw[t];
#pragma unroll
                        for (int k = 1; k >= 0; --k) acc[v][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[v], pf[k], acc[v][t], 0, 0, 0);
#pragma unroll
                        for (int e = 0; e < 4; ++e) ss += acc[v][t][e] * acc[v][t][e];       // columns that pad the size are zero
                    }
                    if (args.finish) {
                        ss += __shfl_xor(ss, 16, 64);
                        ss += __shfl_xor(ss, 32, 64);
                        if (g == 0) squares[wave * kC + 16 * t + n] = ss;
                    }
                }
            }
            // ---- S <- d^n S + sum_j k_j (d^(n-1-j) v_j)^T
            bf16x8_t wf[VT][3];
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                float x[8];
                widen(__builtin_bit_cast(u32x4_t, vf[v]), x);
#pragma unroll
                for (int i = 0; i < 8; ++i) x[i] *= vw[i];
                split_frags<3>(x, wf[v]);
            }
            const unsigned char* kr = kbuf + (8 * g + (n >> 2)) * kRow + (n & 3) * 8;
#pragma unroll
            for (int t = 0; t < 2 * DT; ++t) {
                bf16x8_t kf[PC];
#pragma unroll
                for (int k = 0; k < PC; ++k) {
                    const i16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(kr + k * kMat + 32 * t));
                    const i16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(kr + k * kMat + 32 * t + 4 * kRow));
                    kf[k] = __builtin_bit_cast(bf16x8_t, (i16x8)__builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
                }
#pragma unroll
                for (int v = 0; v < VT; ++v) {
                    s[t][v] *= chunk_decay;
                    s[t][v] = mfma_pieces<3>(kf, wf[v], s[t][v]);
                }
            }
        } else if (OUT && args.finish && lane < kC) {
            squares[wave * kC + lane] = 0.f;
        }
        __syncthreads();
        if constexpr (OUT) {
            // ---- results, with the norm over the head and the gate if nobody else does them
            if (live)
#pragma unroll
                for (int t = 0; t < 2; ++t) {
                    if (16 * t + n >= left) continue;
                    const int64_t row = row0 + c * kC + 16 * t + n;
                    float rs = 1.f;
                    if (args.finish) {
                        float ss = 0.f;
#pragma unroll
                        for (int w = 0; w < 4; ++w) ss += squares[w * kC + 16 * t + n];
                        rs = rsqrtf(ss / (float)a.vdim + args.b.eps);
                    }
#pragma unroll
                    for (int v = 0; v < VT; ++v) {
                        const int col = v0 + 16 * v + 4 * g;
                        if (col >= a.vdim) continue;
                        float x[4];
#pragma unroll
                        for (int e = 0; e < 4; ++e) x[e] = acc[v][t][e];
                        __bf16* o = a.o + row * a.o_stride + (int64_t)h * a.vdim + col;
                        if (args.finish) {
                            const bf16x4_t z = __builtin_bit_cast(bf16x4_t, gate[v][t]);
#pragma unroll
                            for (int e = 0; e < 4; ++e) x[e] *= rs * gate_of(args.b, (float)z[e]);
                            if (args.b.norm)
#pragma unroll
                                for (int e = 0; e < 4; ++e) x[e] *= args.b.norm[h * a.vdim + col + e];
                            o = args.b.out + row * args.b.out_stride + (int64_t)h * a.vdim + col;
                        }
                        store_elems<4>(o, x);
                    }
                }
        }
    }
    if (OUT && !last_seg) return;
#pragma unroll
    for (int t = 0; t < 2 * DT; ++t)
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            const int col = v0 + 16 * v + n;
            if (col < a.vdim_pad)
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (16 * t + 4 * g + e < a.dim_pad) to[(int64_t)(16 * t + 4 * g + e) * a.vdim_pad + col] = s[t][v][e];
        }
}

// ws[span][segment] holds what a segment adds to the state; afterwards the state before the segment
__global__ void __launch_bounds__(kThreads) decay_join_kernel(ChunkArgs args) {
    const DecayArgs<__bf16>& a = args.a;
    const int h = blockIdx.y;
    const Span span = args.spans[blockIdx.z];
    const int64_t state_len = (int64_t)a.dim_pad * a.vdim_pad, i = ((int64_t)blockIdx.x * kThreads + threadIdx.x) * 4;
    if (span.slot < 0 || span.slot >= a.num_slots || i >= state_len) return;
    const float seg_decay = exp2f((float)args.seg_len * a.decay[2 * a.heads + h]);
    f32x4_t s = {0.f, 0.f, 0.f, 0.f};
    if (span.pos0 > 0) s = *reinterpret_cast<const f32x4_t*>(a.state + ((int64_t)span.slot * a.heads + h) * state_len + i);
    for (int seg = 0; seg * args.seg_len < span.count; ++seg) {
        f32x4_t* p = reinterpret_cast<f32x4_t*>(args.ws + (((int64_t)blockIdx.z * args.max_seg + seg) * a.heads + h) * state_len + i);
        f32x4_t add = {0.f, 0.f, 0.f, 0.f};
        if ((seg + 1) * args.seg_len < span.count) add = *p;
        *p = s;
        s = s * seg_decay + add;
    }
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

// sizes the chunk kernel is built for
bool chunks_fit(int elem, int64_t dim, int64_t vdim, int64_t rot_dims) {
    return elem == INFER_ELEM_BF16 && dim % 16 == 0 && vdim % 8 == 0 && dim <= 256 && rot_dims % 16 == 0;
}
int tiles_of(int64_t dim_pad) { return dim_pad <= 32 ? 1 : dim_pad <= 64 ? 2 : dim_pad <= 128 ? 4 : 8; }
int column_tiles(int64_t dim_pad, int64_t vdim_pad) { return vdim_pad <= 64 || dim_pad > 128 ? 1 : 2; }    // per wavefront
int slabs_of(int64_t dim_pad, int64_t vdim_pad) {
    const int cols = 64 * column_tiles(dim_pad, vdim_pad);
    return (int)((vdim_pad + cols - 1) / cols);
}
// tokens per segment: enough segments for two workgroups per compute unit, none shorter than four chunks
int64_t segment_len(int64_t heads, int64_t slabs, int64_t num_spans, int64_t max_span) {
    const int64_t groups = heads * slabs * num_spans;
    int64_t n = (512 + groups - 1) / groups;
    const int64_t most = max_span / (4 * kC);
    if (n > most) n = most;
    if (n <= 1) return (max_span + kC - 1) / kC * kC;
    return ((max_span + n - 1) / n + kC - 1) / kC * kC;
}

template <int DT, int VT, int PC, bool OUT>
int launch_chunk(const ChunkArgs& c, int64_t num_spans, hipStream_t st) {
    const size_t lds = (size_t)kC * ((OUT ? PC == 3 ? 5 : 2 : PC) * (DT * 64 + 16) + 128 * VT + 16) + (OUT ? kC * (2 * (2 * kC + 16) + 16) : 0);
    auto kernel = &decay_chunk_kernel<DT, VT, PC, OUT>;
    if (lds > 64 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return (int)e;
    }
    hipLaunchKernelGGL(kernel, dim3((unsigned)(c.slabs * c.max_seg), (unsigned)c.a.heads, (unsigned)num_spans), dim3(256), lds, st, c);
    return (int)hipGetLastError();
}

template <int DT, int VT>
int launch_chunks(const ChunkArgs& c, int64_t num_spans, hipStream_t st) {
    const bool rot = c.a.rot_pairs > 0;
    int rc;
    if (c.max_seg > 1) {
        rc = rot ? launch_chunk<DT, VT, 3, false>(c, num_spans, st) : launch_chunk<DT, VT, 1, false>(c, num_spans, st);
        if (rc) return rc;
        const unsigned blocks = (unsigned)(((int64_t)c.a.dim_pad * c.a.vdim_pad / 4 + kThreads - 1) / kThreads);
        hipLaunchKernelGGL(decay_join_kernel, dim3(blocks, (unsigned)c.a.heads, (unsigned)num_spans), dim3(kThreads), 0, st, c);
        rc = (int)hipGetLastError();
        if (rc) return rc;
    }
    return rot ? launch_chunk<DT, VT, 3, true>(c, num_spans, st) : launch_chunk<DT, VT, 1, true>(c, num_spans, st);
}

int run_chunks(const ChunkArgs& c, int64_t num_spans, hipStream_t st) {
    const int vt = column_tiles(c.a.dim_pad, c.a.vdim_pad);
    switch (tiles_of(c.a.dim_pad)) {
        case 1: return vt == 1 ? launch_chunks<1, 1>(c, num_spans, st) : launch_chunks<1, 2>(c, num_spans, st);
        case 2: return vt == 1 ? launch_chunks<2, 1>(c, num_spans, st) : launch_chunks<2, 2>(c, num_spans, st);
        case 4: return vt == 1 ? launch_chunks<4, 1>(c, num_spans, st) : launch_chunks<4, 2>(c, num_spans, st);
        default: return launch_chunks<8, 1>(c, num_spans, st);
    }
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

extern "C" int64_t infer_decay_workspace_floats(int elem, int64_t heads, int64_t dim, int64_t vdim, int64_t rot_dims, int64_t num_spans,
                                                int64_t max_span) {
    int64_t pad[2];
    if (infer_decay_layout(dim, vdim, pad) || heads < 1 || num_spans < 1 || max_span < 1 || !chunks_fit(elem, dim, vdim, rot_dims)) return 0;
    const int64_t len = segment_len(heads, slabs_of(pad[0], pad[1]), num_spans, max_span), n = (max_span + len - 1) / len;
    return n > 1 ? num_spans * n * heads * pad[0] * pad[1] : 0;
}

extern "C" int infer_decay_attention(int elem, const void* proj, int64_t proj_stride, int64_t q_off, int64_t k_off, int64_t v_off,
                                     int64_t g_off, int64_t heads, int64_t dim, int64_t vdim, const float* decay, int silu,
                                     const float* table, int64_t rot_dims, int64_t max_pos, float scale, const float* norm,
                                     int norm_per_head, int gate_silu, float eps, float* state, int64_t num_slots,
                                     const int32_t* slots, const int64_t* positions, int64_t decode_rows, const int32_t* spans,
                                     int64_t num_spans, int64_t max_span, int64_t rows, float* workspace, int64_t workspace_floats,
                                     void* out, int64_t out_stride, void* stream) {
    int64_t pad[2];
    if (!size_in(rows, 0, 0x7fffffff) || !size_in(decode_rows, 0, rows) || !size_in(num_spans, 0, 65535)) return INFER_KV_EINVAL;
    if (rows == 0) return INFER_KV_OK;
    if (!proj || !decay || !state || !out || (decode_rows > 0 && (!slots || !positions)) || (decode_rows < rows && (!spans || num_spans < 1 || max_span < 1 || max_span > rows)))
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
        if (decode_rows < rows) {
            bool chunked = false;
            if constexpr (sizeof(T) == 2) {
                chunked = chunks_fit(elem, dim, vdim, rot_dims) && (q_off | k_off | v_off | proj_stride) % 8 == 0 && ptr_aligned(proj, 16) &&
                          out_stride % 4 == 0 && ptr_aligned(out, 8) && ptr_aligned(table, 16);
                if (chunked) {
                    const int slabs = slabs_of(pad[0], pad[1]);
                    const int64_t len = segment_len(heads, slabs, num_spans, max_span), n = (max_span + len - 1) / len;
                    if (n > 1 && (!workspace || !ptr_aligned(workspace, 16) || workspace_floats < num_spans * n * heads * pad[0] * pad[1]))
                        return (int)INFER_KV_EWORKSPACE;
                    // a workgroup that has the whole head norms it, too
                    const bool finish = norm_per_head && slabs == 1 && finished == decode_rows && ptr_aligned(proj, 8) && g_off % 4 == 0;
                    rc = run_chunks(ChunkArgs{a, b, finish, (const Span*)spans, (int)len, (int)n, slabs, workspace}, num_spans, st);
                    if (finish) finished = rows;
                }
            }
            if (!chunked) rc = launch_any(a, (const Span*)spans, nullptr, nullptr, num_spans, st);
        }
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
