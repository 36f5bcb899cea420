// Gated delta rule with a decay per key channel, for gfx950 (MI355X).  Per head, over a float32 state S[dim][vdim]:
//     S <- e^g * S (rows);  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// with k, q unit vectors behind a short causal convolution and silu, g = -exp(A) softplus(a + dt) <= 0.
//
//   delta_step_kernel    one token per sequence (decode): convolution, norms, gates, recurrence, output norm and
//                        output gate in one launch; one workgroup per (sequence, head), the state passes
//                        through registers once
//   delta_prep_kernel    prompt portions in chunks of 16 tokens, all chunks in parallel: convolution, norms,
//                        gates and everything of a chunk that does not need the state
//   delta_scan_kernel    walks the chunks of a portion; a wavefront holds 16 columns of the state as float32 MFMA
//                        accumulators
//   delta_out_kernel     output norm and gate of the scanned tokens; the convolution's tail goes to its ring
//
// Chunk form.  Let G_i be the sum of g over the chunk's tokens up to i, S the state before the chunk.
//     u_i = beta_i (v_i - S^T (e^{G_i} k_i) - sum_{j<i} A_ij u_j),    A_ij = sum_d k_i[d] k_j[d] e^{G_i - G_j}[d]
// so U = T (beta V) - T (beta e^G K) S with T = (I + tril(beta A, -1))^-1, and
//     o_i = (e^{G_i} q_i)^T S + sum_{j<=i} B_ij u_j,                  B_ij = sum_d q_i[d] k_j[d] e^{G_i - G_j}[d]
//     S'  = e^{G_last} S + sum_j (e^{G_last - G_j} k_j) u_j^T.
// Every exponent is a difference that is <= 0, so nothing overflows however strong the decay is.  All of it is
// float32, the products included (v_mfma_f32_16x16x4_f32).
//
// The last `taps` inputs of the convolution live in a ring per sequence (entry position % taps).  A position below
// zero counts as zero and a portion that starts at position 0 starts from a zero state, so a slot needs no clearing
// when another sequence takes it over.
#include "elem.h"

namespace {

constexpr int kC = 16;               // tokens per chunk
constexpr int kStepThreads = 256;

template <class T>
struct DeltaArgs {
    // inputs of a token row: [q: kv_heads x dim | k: kv_heads x dim | v: heads x vdim | ...], columns 0 .. channels - 1
    const T* proj; int64_t proj_stride;
    int beta_off;                                   // column of the write-strength logits in `proj`
    const T* decay; int64_t decay_stride;           // [row][heads * dim]
    const T* gate; int64_t gate_stride;             // [row][heads * vdim]
    const float* conv;                              // [channels][taps]
    const float* a_log; const float* dt_bias; const float* norm;   // [heads], [heads * dim], [vdim]
    T* ring;                                        // [slots][taps][channels]
    float* state;                                   // [slots][heads][dim_pad][vdim_pad]
    int num_slots;
    int heads, kv_heads, dim, vdim, dim_pad, vdim_pad, taps, channels;
    float eps, q_scale;
    T* out; int64_t out_stride;                     // [row][heads * vdim]
};

// silu of the convolution of channel c at position `pos`; row(p) is the batch row of position p >= first, earlier
// positions are in the ring
template <class T, class Row>
__device__ __forceinline__ float conv_silu(const DeltaArgs<T>& a, int c, int64_t pos, int64_t first, int slot, Row row) {
    const float* w = a.conv + (int64_t)c * a.taps;
    float s = 0.f;
    for (int j = 0; j < a.taps; ++j) {
        const int64_t p = pos - j;
        if (p < 0) break;
        const float x = p >= first ? (float)a.proj[row(p) * a.proj_stride + c]
                                   : (float)a.ring[((int64_t)slot * a.taps + p % a.taps) * a.channels + c];
        s += w[a.taps - 1 - j] * x;
    }
    return silu_f(s);
}

template <class T>
__device__ __forceinline__ float log2_decay(const DeltaArgs<T>& a, int64_t row, int h, int d, float rate) {
    const int i = h * a.dim + d;
    return -rate * softplus_f((float)a.decay[row * a.decay_stride + i] + a.dt_bias[i]) * kLog2e;
}

// ------------------------------------------------------------------ one token per sequence
// Thread (r, c): column group c (4 columns of the state), rows r, r + R, ...  NP = rows per thread kept in
// registers; NP = 0: the state is too large for that and is read twice.
template <class T, int NP>
__global__ void __launch_bounds__(kStepThreads) delta_step_kernel(DeltaArgs<T> a, const int32_t* slots, const int64_t* positions) {
    extern __shared__ __attribute__((aligned(16))) float sh[];
    const int row = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    const int slot = slots[row];
    T* out = a.out + (int64_t)row * a.out_stride + (int64_t)h * a.vdim;
    if (slot < 0 || slot >= a.num_slots) {           // a padding row of a captured batch
        for (int v = tid; v < a.vdim; v += kStepThreads) out[v] = (T)0.f;
        return;
    }
    const int64_t pos = positions[row];
    const int group = a.heads / a.kv_heads, kvh = h / group;
    const int cgs = a.vdim_pad / 4, rgs = kStepThreads / cgs;
    float* ks = sh;                                  // [dim_pad]
    float* qs = ks + a.dim_pad;
    float* es = qs + a.dim_pad;                      // e^g
    float* vs = es + a.dim_pad;                      // [vdim_pad]
    float* red = vs + a.vdim_pad;                    // [rgs][vdim_pad]
    float* part = red + rgs * a.vdim_pad;            // [3][4]

    const int cg = tid % cgs, rg = tid / cgs;
    const bool works = rg < rgs;
    float* sp = a.state + (((int64_t)slot * a.heads + h) * a.dim_pad) * a.vdim_pad + 4 * cg;
    f32x4_t s[NP > 0 ? NP : 1];
    if constexpr (NP > 0) {
        if (works)
#pragma unroll
            for (int i = 0; i < NP; ++i) {
                const int d = rg + i * rgs;
                s[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
                if (pos > 0 && d < a.dim_pad) s[i] = *reinterpret_cast<const f32x4_t*>(sp + (int64_t)d * a.vdim_pad);
            }
    }
    auto this_row = [&](int64_t) { return (int64_t)row; };
    const float rate = expf(a.a_log[h]);
    float sk = 0.f, sq = 0.f;
    for (int d = tid; d < a.dim_pad; d += kStepThreads) {
        float k = 0.f, q = 0.f, e = 1.f;
        if (d < a.dim) {
            q = conv_silu(a, kvh * a.dim + d, pos, pos, slot, this_row);
            k = conv_silu(a, (a.kv_heads + kvh) * a.dim + d, pos, pos, slot, this_row);
            e = exp2f(log2_decay(a, row, h, d, rate));
        }
        sk += k * k;
        sq += q * q;
        ks[d] = k; qs[d] = q; es[d] = e;
    }
    for (int v = tid; v < a.vdim_pad; v += kStepThreads)
        vs[v] = v < a.vdim ? conv_silu(a, 2 * a.kv_heads * a.dim + h * a.vdim + v, pos, pos, slot, this_row) : 0.f;
    // The ring holds `taps` entries, one more than the convolution looks back: the entry this token overwrites is
    // not read by anyone, so every workgroup may write its own channels at any time.
    T* ring = a.ring + ((int64_t)slot * a.taps + pos % a.taps) * a.channels;
    const T* in = a.proj + (int64_t)row * a.proj_stride;
    if (h % group == 0)
        for (int d = tid; d < a.dim; d += kStepThreads) {
            ring[kvh * a.dim + d] = in[kvh * a.dim + d];
            ring[(a.kv_heads + kvh) * a.dim + d] = in[(a.kv_heads + kvh) * a.dim + d];
        }
    for (int v = tid; v < a.vdim; v += kStepThreads) {
        const int c = 2 * a.kv_heads * a.dim + h * a.vdim + v;
        ring[c] = in[c];
    }
    const float inv_k = rsqrtf(block_sum<4>(sk, part) + 1e-6f);
    const float inv_q = rsqrtf(block_sum<4>(sq, part + 4) + 1e-6f) * a.q_scale;
    const float beta = sigmoid_f((float)in[a.beta_off + h]);

    // S^T k after the decay
    f32x4_t dot = {0.f, 0.f, 0.f, 0.f};
    if (works) {
        if constexpr (NP > 0) {
#pragma unroll
            for (int i = 0; i < NP; ++i) {
                const int d = rg + i * rgs;
                if (d < a.dim_pad) {
                    s[i] *= es[d];
                    dot += s[i] * ks[d];
                }
            }
        } else if (pos > 0) {
            for (int d = rg; d < a.dim_pad; d += rgs) dot += *reinterpret_cast<const f32x4_t*>(sp + (int64_t)d * a.vdim_pad) * (es[d] * ks[d]);
        }
        *reinterpret_cast<f32x4_t*>(red + rg * a.vdim_pad + 4 * cg) = dot;
    }
    __syncthreads();
    f32x4_t u = {0.f, 0.f, 0.f, 0.f};
    if (works) {
        for (int r = 0; r < rgs; ++r) u += *reinterpret_cast<const f32x4_t*>(red + r * a.vdim_pad + 4 * cg);
        u = (*reinterpret_cast<const f32x4_t*>(vs + 4 * cg) - u * inv_k) * (beta * inv_k);     // k enters as ks * inv_k
    }
    __syncthreads();
    f32x4_t o = {0.f, 0.f, 0.f, 0.f};
    if (works) {
        if constexpr (NP > 0) {
#pragma unroll
            for (int i = 0; i < NP; ++i) {
                const int d = rg + i * rgs;
                if (d < a.dim_pad) {
                    s[i] += u * ks[d];
                    o += s[i] * qs[d];
                    *reinterpret_cast<f32x4_t*>(sp + (int64_t)d * a.vdim_pad) = s[i];
                }
            }
        } else {
            for (int d = rg; d < a.dim_pad; d += rgs) {
                f32x4_t x = {0.f, 0.f, 0.f, 0.f};
                if (pos > 0) x = *reinterpret_cast<const f32x4_t*>(sp + (int64_t)d * a.vdim_pad) * es[d];
                x += u * ks[d];
                o += x * qs[d];
                *reinterpret_cast<f32x4_t*>(sp + (int64_t)d * a.vdim_pad) = x;
            }
        }
        *reinterpret_cast<f32x4_t*>(red + rg * a.vdim_pad + 4 * cg) = o * inv_q;
    }
    __syncthreads();
    // vdim_pad <= 1024 = 4 column groups of threads; one thread per column group finishes the row
    float so = 0.f;
    f32x4_t y = {0.f, 0.f, 0.f, 0.f};
    if (tid < cgs) {
        for (int r = 0; r < rgs; ++r) y += *reinterpret_cast<const f32x4_t*>(red + r * a.vdim_pad + 4 * tid);
#pragma unroll
        for (int e = 0; e < 4; ++e) so += y[e] * y[e];       // padded columns are zero
    }
    const float rs = rsqrtf(block_sum<4>(so, part + 8) / (float)a.vdim + a.eps);
    if (tid < cgs) {
        const T* gr = a.gate + (int64_t)row * a.gate_stride + (int64_t)h * a.vdim;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int v = 4 * tid + e;
            if (v < a.vdim) out[v] = (T)(y[e] * rs * a.norm[v] * sigmoid_f((float)gr[v]));
        }
    }
}

// ------------------------------------------------------------------ prompt portions
struct ChunkDesc { int32_t row0, count, pos0, first_pos, slot, pad; };   // first_pos: where the portion starts
struct PortionDesc { int32_t chunk0, chunks, slot, pos0; };

// A chunk's record, floats, each part in the order in which the lanes of the scan read it (lane = 16 q + m takes the
// four consecutive floats at 4 * lane of a 256-float fragment):
//   W   [dim_pad / 16][256]   element (i, d):  T (beta e^G K)
//   Q   [dim_pad / 16][256]   element (i, d):  e^G q
//   K   [dim_pad / 16][256]   element (j, d):  e^{G_last - G_j} k_j, rows d
//   B   [256]                 element (i, j)
//   E   [dim_pad]             e^{G_last}
//   V   [vdim_pad / 16][256]  element (i, v):  T (beta V)
__host__ __device__ inline int64_t record_floats(int dim_pad, int vdim_pad) { return 48 * (int64_t)dim_pad + 256 + dim_pad + 16 * (int64_t)vdim_pad; }

// The convolution of four channels over tokens t0 .. t0 + 7 of a chunk, for four taps, the window in registers.
// c: first channel, dst: LDS row of token t0, column of the channel.  INNER: all 16 tokens exist and the window of
// the first one lies inside the portion.
template <class T, bool INNER>
__device__ __forceinline__ void conv4_silu(const DeltaArgs<T>& a, const ChunkDesc& cd, int c, int t0, float* dst, int pitch) {
    float x[11][4], w[4][4];
#pragma unroll
    for (int e = 0; e < 4; ++e) load_elems<4>(a.conv + 4 * (c + e), w[e]);
    if constexpr (INNER) {
        const T* src = a.proj + (int64_t)(cd.row0 + t0 - 3) * a.proj_stride + c;
#pragma unroll
        for (int j = 0; j < 11; ++j, src += a.proj_stride) load_elems<4>(src, x[j]);
    }
#pragma unroll
    for (int j = 0; j < (INNER ? 0 : 11); ++j) {
        const int t = t0 + j - 3, p = cd.pos0 + t;
        // positions before the portion are in the ring; those before the sequence or behind the chunk's tokens are zero
        const bool in = p >= 0 && t < cd.count;
        const T* src = p >= cd.first_pos || !in ? a.proj + (int64_t)(cd.row0 + (in ? t : 0)) * a.proj_stride + c
                                                : a.ring + ((int64_t)cd.slot * 4 + (p & 3)) * a.channels + c;
        load_elems<4>(src, x[j]);
        if (!in)
#pragma unroll
            for (int e = 0; e < 4; ++e) x[j][e] = 0.f;
    }
#pragma unroll
    for (int t = 0; t < 8; ++t) {
        float y[4];
        const bool in = INNER || t0 + t < cd.count;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            y[e] = 0.f;
#pragma unroll
            for (int j = 0; j < 4; ++j) y[e] += w[e][j] * x[t + j][e];
            y[e] = in ? silu_f(y[e]) : 0.f;
        }
        store_elems<4>(dst + t * pitch, y);
    }
}

// softplus in units of log2: log2(1 + e^z)
__device__ __forceinline__ float softplus_log2(float z) {
    const float e = __builtin_amdgcn_exp2f(-fabsf(z) * kLog2e);
    const float l = e < 0.02f ? e * (1.f - e * (0.5f - e * (0.33333333f - 0.25f * e))) * kLog2e : __builtin_amdgcn_logf(1.f + e);
    return fmaxf(z, 0.f) * kLog2e + l;
}

// Decay of a whole chunk, in log2 units, up to which e^{G_i - G_j} may be split into two factors.
constexpr float kSplitRange = 48.f;

// VEC: four channels at a time, four taps; otherwise any size, one element at a time.
template <class T, bool VEC>
__global__ void __launch_bounds__(256) delta_prep_kernel(DeltaArgs<T> a, const ChunkDesc* chunks, float* records) {
    extern __shared__ __attribute__((aligned(16))) float sh[];
    const int tid = threadIdx.x, h = blockIdx.y, lane = tid & 63, wave = tid >> 6;
    const ChunkDesc c = chunks[blockIdx.x];
    const int dp = a.dim_pad, pk = dp + 4, pv = a.vdim_pad + 4;
    float* qs = sh;                    // [16][pk] q, then e^G q
    float* ks = qs + kC * pk;          // [16][pk] k, then e^G k
    float* gs = ks + kC * pk;          // [16][pk] running log2 decay G, then e^{G_last - G} k
    float* vs = gs + kC * pk;          // [16][pv]
    float* pp = vs + kC * pv;          // [2][2][256] products of the token pairs (k k, q k), in two parts each
    float* lt = pp + 1024;             // [16][20] column s: beta * A of the tokens behind s
    float* tb = lt;                    // [16][20] T * beta, when those have been used
    float* gl = lt + kC * 20;          // [dp] G_last
    float* inv = gl + dp;              // [2][16] 1 / length of k and q
    float* bs = inv + 32;              // [16] beta
    const int group = a.heads / a.kv_heads, kvh = h / group;
    const int cq = kvh * a.dim, ck = (a.kv_heads + kvh) * a.dim, cv = 2 * a.kv_heads * a.dim + h * a.vdim;
    float* rec = records + ((int64_t)blockIdx.x * a.heads + h) * record_floats(dp, a.vdim_pad);
    const float rate = expf(a.a_log[h]);

    if constexpr (VEC) {
        const int nd = a.dim / 4, nv = a.vdim / 4, n = 2 * nd + nv;
        const bool inner = c.count == kC && c.pos0 - 3 >= c.first_pos;
        for (int i = tid; i < 2 * n; i += 256) {
            const int half = i >= n, j = i - half * n, t0 = 8 * half;
            const int col = j < nd ? 4 * j : j < 2 * nd ? 4 * (j - nd) : 4 * (j - 2 * nd);
            const int ch = col + (j < nd ? cq : j < 2 * nd ? ck : cv), pitch = j < 2 * nd ? pk : pv;
            float* dst = (j < nd ? qs : j < 2 * nd ? ks : vs) + t0 * pitch + col;
            if (inner) conv4_silu<T, true>(a, c, ch, t0, dst, pitch);
            else conv4_silu<T, false>(a, c, ch, t0, dst, pitch);
        }
        for (int i = tid; i < kC * nd; i += 256) {
            const int t = i / nd, d = 4 * (i - t * nd);
            float x[4] = {0.f, 0.f, 0.f, 0.f};
            if (t < c.count) {
                float dt[4];
                load_elems<4>(a.decay + (int64_t)(c.row0 + t) * a.decay_stride + h * a.dim + d, x);
                load_elems<4>(a.dt_bias + h * a.dim + d, dt);
#pragma unroll
                for (int e = 0; e < 4; ++e) x[e] = -rate * softplus_log2(x[e] + dt[e]);
            }
            store_elems<4>(gs + t * pk + d, x);
        }
        for (int i = tid; i < kC * (dp - a.dim); i += 256) {
            const int t = i / (dp - a.dim), d = a.dim + i % (dp - a.dim);
            qs[t * pk + d] = ks[t * pk + d] = gs[t * pk + d] = 0.f;
        }
        for (int i = tid; i < kC * (a.vdim_pad - a.vdim); i += 256) {
            const int t = i / (a.vdim_pad - a.vdim), v = a.vdim + i % (a.vdim_pad - a.vdim);
            vs[t * pv + v] = 0.f;
        }
    } else {
        auto row_of = [&](int64_t p) { return (int64_t)c.row0 + (p - c.pos0); };
        for (int i = tid; i < kC * dp; i += 256) {
            const int t = i / dp, d = i - t * dp;
            float q = 0.f, k = 0.f, g = 0.f;
            if (t < c.count && d < a.dim) {
                q = conv_silu(a, cq + d, c.pos0 + t, c.first_pos, c.slot, row_of);
                k = conv_silu(a, ck + d, c.pos0 + t, c.first_pos, c.slot, row_of);
                g = log2_decay(a, c.row0 + t, h, d, rate);
            }
            qs[t * pk + d] = q;
            ks[t * pk + d] = k;
            gs[t * pk + d] = g;
        }
        for (int i = tid; i < kC * a.vdim_pad; i += 256) {
            const int t = i / a.vdim_pad, v = i - t * a.vdim_pad;
            vs[t * pv + v] = t < c.count && v < a.vdim ? conv_silu(a, cv + v, c.pos0 + t, c.first_pos, c.slot, row_of) : 0.f;
        }
    }
    if (tid < kC) bs[tid] = tid < c.count ? sigmoid_f((float)a.proj[(int64_t)(c.row0 + tid) * a.proj_stride + a.beta_off + h]) : 0.f;
    __syncthreads();

    const int i = tid >> 4, j = tid & 15;
    int strong = 0;
    for (int d = tid; d < dp; d += 256) {
        float sum = 0.f;
#pragma unroll
        for (int t = 0; t < kC; ++t) {
            sum += gs[t * pk + d];
            gs[t * pk + d] = sum;
        }
        gl[d] = sum;
        strong |= sum < -kSplitRange;
    }
    {
        float sk = 0.f, sq = 0.f;
        for (int d = 4 * j; d < dp; d += 64) {
            const f32x4_t k = *reinterpret_cast<const f32x4_t*>(ks + i * pk + d), q = *reinterpret_cast<const f32x4_t*>(qs + i * pk + d);
#pragma unroll
            for (int e = 0; e < 4; ++e) { sk += k[e] * k[e]; sq += q[e] * q[e]; }
        }
#pragma unroll
        for (int m = 8; m >= 1; m >>= 1) { sk += __shfl_xor(sk, m, 64); sq += __shfl_xor(sq, m, 64); }
        if (j == 0) { inv[i] = rsqrtf(sk + 1e-6f); inv[16 + i] = rsqrtf(sq + 1e-6f) * a.q_scale; }
    }
    strong = __syncthreads_or(strong);
    float akk = 0.f, aqk = 0.f;                    // products of token pair (i, j), before the lengths
    if (strong && j <= i) {
        // some channel decays so much over the chunk that only differences of G can be exponentiated
        const float *ki = ks + i * pk, *qi = qs + i * pk, *gi = gs + i * pk, *kj = ks + j * pk, *gj = gs + j * pk;
        for (int d = 0; d < dp; d += 4) {
            const f32x4_t k1 = *reinterpret_cast<const f32x4_t*>(ki + d), q1 = *reinterpret_cast<const f32x4_t*>(qi + d);
            const f32x4_t g1 = *reinterpret_cast<const f32x4_t*>(gi + d), k2 = *reinterpret_cast<const f32x4_t*>(kj + d);
            const f32x4_t g2 = *reinterpret_cast<const f32x4_t*>(gj + d);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float w = k2[e] * __builtin_amdgcn_exp2f(g1[e] - g2[e]);
                akk += k1[e] * w;
                aqk += q1[e] * w;
            }
        }
    }
    if (strong) __syncthreads();
    for (int x = tid; x < kC * (dp / 4); x += 256) {
        const int t = x / (dp / 4), d = 4 * (x - t * (dp / 4));
        f32x4_t* g = reinterpret_cast<f32x4_t*>(gs + t * pk + d);
        f32x4_t* k = reinterpret_cast<f32x4_t*>(ks + t * pk + d);
        f32x4_t* q = reinterpret_cast<f32x4_t*>(qs + t * pk + d);
        const f32x4_t last = *reinterpret_cast<const f32x4_t*>(gl + d);
        f32x4_t gv = *g, kv = *k, qv = *q;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const float up = __builtin_amdgcn_exp2f(gv[e]);
            gv[e] = kv[e] * __builtin_amdgcn_exp2f(last[e] - gv[e]);
            kv[e] *= up;
            qv[e] *= up;
        }
        *g = gv; *k = kv; *q = qv;
    }
    __syncthreads();
    const int lq = lane >> 4, lm = lane & 15;
    if (!strong) {
        // A_ij = sum_d (k_i e^{G_i - G_last}) (k_j e^{G_last - G_j}) on the matrix pipe: wavefronts 0 and 1 take half of the
        // channels each, 2 and 3 do the same for q
        f32x4_t acc0 = {0.f, 0.f, 0.f, 0.f}, acc1 = acc0;
        const float* left = (wave < 2 ? ks : qs) + lm * pk;
        for (int t = wave & 1; t < dp / 16; t += 2) {
            const int d = 16 * t + 4 * lq;
            const f32x4_t x1 = *reinterpret_cast<const f32x4_t*>(left + d), last = *reinterpret_cast<const f32x4_t*>(gl + d);
            const f32x4_t k2 = *reinterpret_cast<const f32x4_t*>(gs + lm * pk + d);
#pragma unroll
            for (int e = 0; e < 4; e += 2) {
                acc0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x1[e] * __builtin_amdgcn_exp2f(-last[e]), k2[e], acc0, 0, 0, 0);
                acc1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x1[e + 1] * __builtin_amdgcn_exp2f(-last[e + 1]), k2[e + 1], acc1, 0, 0, 0);
            }
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) pp[wave * 256 + (4 * lq + e) * 16 + lm] = acc0[e] + acc1[e];    // row: token i, column: token j
        __syncthreads();
        akk = pp[tid] + pp[256 + tid];
        aqk = pp[512 + tid] + pp[768 + tid];
    }
    lt[j * 20 + i] = j < i ? bs[i] * akk * inv[i] * inv[j] : 0.f;
    rec[48 * dp + ((j >> 2) * 16 + i) * 4 + (j & 3)] = j <= i ? aqk * inv[16 + i] * inv[j] : 0.f;
    __syncthreads();
    if (wave == 0) {
        // T = (I + L)^-1 column by column: lane m holds column m, row s is final when it is used
        float t[kC];
#pragma unroll
        for (int r = 0; r < kC; ++r) t[r] = r == lm ? 1.f : 0.f;
#pragma unroll
        for (int s = 0; s < kC - 1; ++s)
#pragma unroll
            for (int r4 = 0; r4 < kC; r4 += 4)
                if (r4 + 3 > s) {
                    const f32x4_t l = *reinterpret_cast<const f32x4_t*>(lt + s * 20 + r4);      // zero for rows up to s
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (r4 + e > s) t[r4 + e] -= l[e] * t[s];
                }
        if (lane < kC) {
            const float b = bs[lm];
#pragma unroll
            for (int r = 0; r < kC; ++r) tb[r * 20 + lm] = t[r] * b;
        }
    } else {
        const float iq = inv[16 + lm];
        f32x4_t ik;
#pragma unroll
        for (int e = 0; e < 4; ++e) ik[e] = inv[4 * lq + e];
        for (int t = wave - 1; t < dp / 16; t += 3) {
            f32x4_t q = *reinterpret_cast<const f32x4_t*>(qs + lm * pk + 16 * t + 4 * lq), k;
            q *= iq;
#pragma unroll
            for (int e = 0; e < 4; ++e) k[e] = gs[(4 * lq + e) * pk + 16 * t + lm] * ik[e];
            *reinterpret_cast<f32x4_t*>(rec + 16 * dp + 256 * t + 4 * lane) = q;
            *reinterpret_cast<f32x4_t*>(rec + 32 * dp + 256 * t + 4 * lane) = k;
        }
        for (int d = tid - 64; d < dp; d += 192) rec[48 * dp + 256 + d] = __builtin_amdgcn_exp2f(gl[d]);
    }
    __syncthreads();
    const f32x4_t tv = *reinterpret_cast<const f32x4_t*>(tb + lm * 20 + 4 * lq);       // T beta, row lm
    for (int t = wave; t < dp / 16; t += 4) {      // W^T = (e^G K)^T (T beta)^T: row d, column i
        f32x4_t w = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int e = 0; e < 4; ++e)
            w = __builtin_amdgcn_mfma_f32_16x16x4f32(ks[(4 * lq + e) * pk + 16 * t + lm] * inv[4 * lq + e], tv[e], w, 0, 0, 0);
        *reinterpret_cast<f32x4_t*>(rec + 256 * t + 4 * lane) = w;
    }
    float* uv = rec + 49 * dp + 256;
    for (int t = wave; t < a.vdim_pad / 16; t += 4) {
        f32x4_t w = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int e = 0; e < 4; ++e) w = __builtin_amdgcn_mfma_f32_16x16x4f32(tv[e], vs[(4 * lq + e) * pv + 16 * t + lm], w, 0, 0, 0);
        *reinterpret_cast<f32x4_t*>(uv + 256 * t + 4 * lane) = w;
    }
}

// Wavefront w of workgroup x owns state columns 16 (x * waves + w) .. + 15: DT accumulator tiles of 16 rows, lane (q, m)
// holding rows 16 t + 4 q + r of column m.  That is also the layout of the second operand of the next product, whose
// first operand the records hold in fragment order.
template <int DT>
__global__ void __launch_bounds__(256) delta_scan_kernel(const PortionDesc* portions, const ChunkDesc* chunks, const float* records,
                                                         float* state, float* o, int heads, int vdim_pad) {
    constexpr int dp = 16 * DT;
    constexpr int kShared = 48 * dp + 256 + dp;                  // floats of a record all wavefronts read
    extern __shared__ __attribute__((aligned(16))) float sh[];   // [2][kShared]
    const int tid = threadIdx.x, threads = blockDim.x, lane = tid & 63, wave = tid >> 6;
    const int q = lane >> 4, m = lane & 15;
    const int h = blockIdx.y;
    const PortionDesc p = portions[blockIdx.z];
    const int vt = blockIdx.x * (threads >> 6) + wave;
    const bool live = vt < vdim_pad / 16;
    const int64_t rec_len = record_floats(dp, vdim_pad);
    float* sp = state + (((int64_t)p.slot * heads + h) * dp) * vdim_pad + 16 * vt + m;
    f32x4_t s[DT];
#pragma unroll
    for (int t = 0; t < DT; ++t) {
        s[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        if (live && p.pos0 > 0)
#pragma unroll
            for (int r = 0; r < 4; ++r) s[t][r] = sp[(int64_t)(16 * t + 4 * q + r) * vdim_pad];
    }
    constexpr int kVecs = kShared / 4;
    constexpr int kMaxStage = (kVecs + 63) / 64;                 // chunks of 16 bytes per thread of a one-wavefront workgroup
    constexpr int kStage = kMaxStage < 8 ? kMaxStage : 8;        // kept in registers; the rest goes straight to LDS
    f32x4_t stage[kStage];
    auto fetch = [&](int c) {
        const f32x4_t* src = reinterpret_cast<const f32x4_t*>(records + ((int64_t)(p.chunk0 + c) * heads + h) * rec_len);
#pragma unroll
        for (int i = 0; i < kStage; ++i)
            if (tid + i * threads < kVecs) stage[i] = src[tid + i * threads];
    };
    auto put = [&](int c, float* buf) {
        f32x4_t* dst = reinterpret_cast<f32x4_t*>(buf);
#pragma unroll
        for (int i = 0; i < kStage; ++i)
            if (tid + i * threads < kVecs) dst[tid + i * threads] = stage[i];
        const f32x4_t* src = reinterpret_cast<const f32x4_t*>(records + ((int64_t)(p.chunk0 + c) * heads + h) * rec_len);
        for (int i = tid + kStage * threads; i < kVecs; i += threads) dst[i] = src[i];
    };
    fetch(0);
    put(0, sh);
    __syncthreads();
    for (int c = 0; c < p.chunks; ++c) {
        const float* buf = sh + (c & 1) * kShared;
        const float* rec = records + ((int64_t)(p.chunk0 + c) * heads + h) * rec_len;
        f32x4_t u = {0.f, 0.f, 0.f, 0.f};
        if (live) u = *reinterpret_cast<const f32x4_t*>(rec + kShared + vt * 256 + 4 * lane);
        if (c + 1 < p.chunks) fetch(c + 1);
        const float* fr = buf + 4 * lane;
        f32x4_t ws0 = {0.f, 0.f, 0.f, 0.f}, ws1 = ws0, o0 = ws0, o1 = ws0;
#pragma unroll
        for (int t = 0; t < DT; ++t) {
            const f32x4_t w = *reinterpret_cast<const f32x4_t*>(fr + 256 * t);
            const f32x4_t qv = *reinterpret_cast<const f32x4_t*>(fr + 16 * dp + 256 * t);
#pragma unroll
            for (int r = 0; r < 4; r += 2) {
                ws0 = __builtin_amdgcn_mfma_f32_16x16x4f32(w[r], s[t][r], ws0, 0, 0, 0);
                o0 = __builtin_amdgcn_mfma_f32_16x16x4f32(qv[r], s[t][r], o0, 0, 0, 0);
                ws1 = __builtin_amdgcn_mfma_f32_16x16x4f32(w[r + 1], s[t][r + 1], ws1, 0, 0, 0);
                o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(qv[r + 1], s[t][r + 1], o1, 0, 0, 0);
            }
        }
        u = u - (ws0 + ws1);
        const f32x4_t b = *reinterpret_cast<const f32x4_t*>(fr + 48 * dp);
#pragma unroll
        for (int r = 0; r < 4; ++r) o0 = __builtin_amdgcn_mfma_f32_16x16x4f32(b[r], u[r], o0, 0, 0, 0);
        const float* e = buf + 48 * dp + 256 + 4 * q;
#pragma unroll
        for (int t = 0; t < DT; ++t) {
            const f32x4_t k = *reinterpret_cast<const f32x4_t*>(fr + 32 * dp + 256 * t);
            s[t] *= *reinterpret_cast<const f32x4_t*>(e + 16 * t);
#pragma unroll
            for (int r = 0; r < 4; ++r) s[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(k[r], u[r], s[t], 0, 0, 0);
        }
        if (live) {
            const ChunkDesc d = chunks[p.chunk0 + c];
            const f32x4_t ov = o0 + o1;
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (4 * q + r < d.count) o[((int64_t)(d.row0 + 4 * q + r) * heads + h) * vdim_pad + 16 * vt + m] = ov[r];
        }
        if (c + 1 < p.chunks) put(c + 1, sh + ((c + 1) & 1) * kShared);
        __syncthreads();
    }
    if (live)
#pragma unroll
        for (int t = 0; t < DT; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) sp[(int64_t)(16 * t + 4 * q + r) * vdim_pad] = s[t][r];
}

// One workgroup per token row behind `row0`.  LANES lanes share a head, four values each (vdim = 4 LANES);
// LANES = 0: any vdim, one wavefront per head.
template <class T, int LANES>
__global__ void __launch_bounds__(256) delta_out_kernel(DeltaArgs<T> a, const float* o, int64_t row0, const int32_t* ring_slot,
                                                        const int64_t* positions) {
    const int64_t row = row0 + blockIdx.x;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    if constexpr (LANES > 0) {
        const int v = 4 * (threadIdx.x % LANES);
        float w[4];
        load_elems<4>(a.norm + v, w);
        for (int h = threadIdx.x / LANES; h < a.heads; h += 256 / LANES) {
            float x[4], g[4];
            load_elems<4>(o + (row * a.heads + h) * a.vdim_pad + v, x);
            load_elems<4>(a.gate + row * a.gate_stride + (int64_t)h * a.vdim + v, g);
            float ss = x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
#pragma unroll
            for (int m = LANES / 2; m >= 1; m >>= 1) ss += __shfl_xor(ss, m, 64);
            const float rs = rsqrtf(ss / (float)a.vdim + a.eps);
#pragma unroll
            for (int e = 0; e < 4; ++e) x[e] *= rs * w[e] * sigmoid_f(g[e]);
            store_elems<4>(a.out + row * a.out_stride + (int64_t)h * a.vdim + v, x);
        }
    } else {
        for (int h = wave; h < a.heads; h += 4) {
            const float* x = o + (row * a.heads + h) * a.vdim_pad;
            float ss = 0.f;
            for (int v = lane; v < a.vdim; v += 64) ss += x[v] * x[v];
            const float rs = rsqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
            const T* gr = a.gate + row * a.gate_stride + (int64_t)h * a.vdim;
            T* out = a.out + row * a.out_stride + (int64_t)h * a.vdim;
            for (int v = lane; v < a.vdim; v += 64) out[v] = (T)(x[v] * rs * a.norm[v] * sigmoid_f((float)gr[v]));
        }
    }
    const int slot = ring_slot[2 * row];
    if (slot < 0 || slot >= a.num_slots || ring_slot[2 * row + 1] >= a.taps) return;     // not among the portion's last inputs
    T* ring = a.ring + ((int64_t)slot * a.taps + positions[row] % a.taps) * a.channels;
    const T* in = a.proj + row * a.proj_stride;
    for (int c = threadIdx.x; c < a.channels; c += 256) ring[c] = in[c];
}

int tiles_of(int dim) {        // row tiles of the state, rounded up to what the scan is built for
    const int t = (dim + 15) / 16;
    for (int n : {1, 2, 3, 4, 6, 8, 12, 16})
        if (t <= n) return n;
    return 0;
}

template <int DT>
int launch_scan(const PortionDesc* p, int64_t portions, const ChunkDesc* c, const float* records, float* state, float* o,
                int heads, int vdim_pad, hipStream_t st) {
    const int slabs = vdim_pad / 16, waves = slabs < 4 ? slabs : 4;
    constexpr size_t lds = (size_t)2 * (49 * 16 * DT + 256) * sizeof(float);
    if (lds > 64 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&delta_scan_kernel<DT>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return (int)e;
    }
    hipLaunchKernelGGL((delta_scan_kernel<DT>), dim3((unsigned)((slabs + waves - 1) / waves), (unsigned)heads, (unsigned)portions),
                       dim3(64 * waves), lds, st, p, c, records, state, o, heads, vdim_pad);
    return (int)hipGetLastError();
}

template <class T>
int make_args(DeltaArgs<T>& a, const void* proj, int64_t proj_stride, int64_t beta_off, const void* decay, int64_t decay_stride,
              const void* gate, int64_t gate_stride, const float* conv, const float* a_log, const float* dt_bias, const float* norm,
              void* ring, float* state, int64_t num_slots, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim, int64_t taps,
              float eps, void* out, int64_t out_stride) {
    if (!proj || !decay || !gate || !conv || !a_log || !dt_bias || !norm || !ring || !state || !out) return INFER_KV_EINVAL;
    if (heads < 1 || heads > 65535 || kv_heads < 1 || heads % kv_heads || dim < 1 || vdim < 1 || taps < 1 || taps > 64 || num_slots < 1 ||
        num_slots > (1 << 24))
        return INFER_KV_EINVAL;
    if (dim > 256 || vdim > 512) return INFER_KV_EUNSUPPORTED;
    const int64_t channels = 2 * kv_heads * dim + heads * vdim;
    if (beta_off < channels || proj_stride < beta_off + heads || decay_stride < heads * dim || gate_stride < heads * vdim ||
        out_stride < heads * vdim)
        return INFER_KV_EINVAL;
    if (!ptr_aligned(state, 16)) return INFER_KV_EALIGN;
    a = DeltaArgs<T>{(const T*)proj, proj_stride, (int)beta_off, (const T*)decay, decay_stride, (const T*)gate, gate_stride, conv, a_log,
                     dt_bias, norm, (T*)ring, state, (int)num_slots, (int)heads, (int)kv_heads, (int)dim, (int)vdim,
                     16 * tiles_of((int)dim), (int)((vdim + 15) / 16 * 16), (int)taps, (int)channels, eps, 1.0f / sqrtf((float)dim),
                     (T*)out, out_stride};
    return INFER_KV_OK;
}

template <class T>
int launch_step(const DeltaArgs<T>& a, const int32_t* slots, const int64_t* positions, int64_t rows, hipStream_t st) {
    const int cgs = a.vdim_pad / 4, rgs = kStepThreads / cgs, np = (a.dim_pad + rgs - 1) / rgs;
    const size_t lds = (size_t)(3 * a.dim_pad + a.vdim_pad + rgs * a.vdim_pad + 12) * sizeof(float);
    const dim3 grid((unsigned)rows, (unsigned)a.heads), block(kStepThreads);
#define GO(N) hipLaunchKernelGGL((delta_step_kernel<T, N>), grid, block, lds, st, a, slots, positions)
    if (np <= 1) GO(1);
    else if (np <= 2) GO(2);
    else if (np <= 4) GO(4);
    else if (np <= 8) GO(8);
    else if (np <= 16) GO(16);
    else if (np <= 32) GO(32);
    else GO(0);
#undef GO
    return (int)hipGetLastError();
}

template <class T>
int launch_chunks(const DeltaArgs<T>& a, const PortionDesc* portions, int64_t num_portions, const ChunkDesc* chunks, int64_t num_chunks,
                  float* records, float* o, int64_t row0, int64_t rows, const int32_t* ring_slot, const int64_t* positions,
                  hipStream_t st) {
    const size_t lds = (size_t)(3 * kC * (a.dim_pad + 4) + kC * (a.vdim_pad + 4) + 1024 + kC * 20 + a.dim_pad + 48) * sizeof(float);
    // rows and channels that can be read four elements at a time
    auto fours = [](const void* p, int64_t stride) { return ptr_aligned(p, 4 * sizeof(T)) && stride % 4 == 0; };
    const bool rows4 = a.dim % 4 == 0 && a.vdim % 4 == 0;
    const bool vec = rows4 && a.taps == 4 && fours(a.proj, a.proj_stride) && fours(a.ring, a.channels) && fours(a.decay, a.decay_stride) &&
                     ptr_aligned(a.conv, 16) && ptr_aligned(a.dt_bias, 16);
    auto prep = vec ? &delta_prep_kernel<T, true> : &delta_prep_kernel<T, false>;
    if (lds > 60 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(prep), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return (int)e;
    }
    hipLaunchKernelGGL(prep, dim3((unsigned)num_chunks, (unsigned)a.heads), dim3(256), lds, st, a, chunks, records);
    int rc = (int)hipGetLastError();
    if (rc) return rc;
#define GO(N) case N: rc = launch_scan<N>(portions, num_portions, chunks, records, a.state, o, a.heads, a.vdim_pad, st); break
    switch (a.dim_pad / 16) { GO(1); GO(2); GO(3); GO(4); GO(6); GO(8); GO(12); GO(16); default: return INFER_KV_EUNSUPPORTED; }
#undef GO
    if (rc) return rc;
    const bool out4 = rows4 && fours(a.gate, a.gate_stride) && fours(a.out, a.out_stride) && ptr_aligned(o, 16) && ptr_aligned(a.norm, 16);
#define GO(N) hipLaunchKernelGGL((delta_out_kernel<T, N>), dim3((unsigned)rows), dim3(256), 0, st, a, (const float*)o, row0, ring_slot, positions)
    if (out4 && a.vdim == 32) GO(8);
    else if (out4 && a.vdim == 64) GO(16);
    else if (out4 && a.vdim == 128) GO(32);
    else if (out4 && a.vdim == 256) GO(64);
    else GO(0);
#undef GO
    return (int)hipGetLastError();
}

}  // namespace

// [0]: state rows per head, [1]: state columns per head, [2]: floats of a chunk record, [3]: tokens per chunk;
// 0 if the sizes are served, otherwise a negative code
extern "C" int infer_delta_layout(int64_t dim, int64_t vdim, int64_t* out4) {
    if (!out4 || dim < 1 || vdim < 1) return INFER_KV_EINVAL;
    if (dim > 256 || vdim > 512) return INFER_KV_EUNSUPPORTED;
    const int dp = 16 * tiles_of((int)dim), vp = (int)((vdim + 15) / 16 * 16);
    out4[0] = dp; out4[1] = vp; out4[2] = record_floats(dp, vp); out4[3] = kC;
    return INFER_KV_OK;
}

extern "C" int infer_delta_step(int elem, const void* proj, int64_t proj_stride, int64_t beta_off, const void* decay,
                                int64_t decay_stride, const void* gate, int64_t gate_stride, const float* conv, const float* a_log,
                                const float* dt_bias, const float* norm, void* ring, float* state, int64_t num_slots, int64_t heads,
                                int64_t kv_heads, int64_t dim, int64_t vdim, int64_t taps, float eps, const int32_t* slots,
                                const int64_t* positions, void* out, int64_t out_stride, int64_t rows, void* stream) {
    if (rows < 0 || rows > 0x7fffffff) return INFER_KV_EINVAL;
    if (rows == 0) return INFER_KV_OK;
    if (!slots || !positions) return INFER_KV_EINVAL;
    int rc;
    if (elem == INFER_ELEM_BF16) {
        DeltaArgs<__bf16> a;
        rc = make_args(a, proj, proj_stride, beta_off, decay, decay_stride, gate, gate_stride, conv, a_log, dt_bias, norm, ring, state,
                       num_slots, heads, kv_heads, dim, vdim, taps, eps, out, out_stride);
        return rc ? rc : launch_step(a, slots, positions, rows, (hipStream_t)stream);
    }
    if (elem == INFER_ELEM_F32) {
        DeltaArgs<float> a;
        rc = make_args(a, proj, proj_stride, beta_off, decay, decay_stride, gate, gate_stride, conv, a_log, dt_bias, norm, ring, state,
                       num_slots, heads, kv_heads, dim, vdim, taps, eps, out, out_stride);
        return rc ? rc : launch_step(a, slots, positions, rows, (hipStream_t)stream);
    }
    return INFER_KV_EUNSUPPORTED;
}

extern "C" int infer_delta_chunks(int elem, const void* proj, int64_t proj_stride, int64_t beta_off, const void* decay,
                                  int64_t decay_stride, const void* gate, int64_t gate_stride, const float* conv, const float* a_log,
                                  const float* dt_bias, const float* norm, void* ring, float* state, int64_t num_slots, int64_t heads,
                                  int64_t kv_heads, int64_t dim, int64_t vdim, int64_t taps, float eps, const int32_t* portions,
                                  int64_t num_portions, const int32_t* chunks, int64_t num_chunks, float* records, float* o,
                                  const int32_t* ring_slot, const int64_t* positions, void* out, int64_t out_stride, int64_t row0,
                                  int64_t rows, void* stream) {
    if (rows < 0 || rows > 0x7fffffff || row0 < 0 || num_portions < 0 || num_portions > 65535 || num_chunks < num_portions ||
        num_chunks > 0x7fffffff)
        return INFER_KV_EINVAL;
    if (rows == 0 || num_portions == 0) return INFER_KV_OK;
    if (!portions || !chunks || !records || !o || !ring_slot || !positions) return INFER_KV_EINVAL;
    if (!ptr_aligned(records, 16)) return INFER_KV_EALIGN;
    int rc;
    if (elem == INFER_ELEM_BF16) {
        DeltaArgs<__bf16> a;
        rc = make_args(a, proj, proj_stride, beta_off, decay, decay_stride, gate, gate_stride, conv, a_log, dt_bias, norm, ring, state,
                       num_slots, heads, kv_heads, dim, vdim, taps, eps, out, out_stride);
        return rc ? rc : launch_chunks(a, (const PortionDesc*)portions, num_portions, (const ChunkDesc*)chunks, num_chunks, records, o,
                                       row0, rows, ring_slot, positions, (hipStream_t)stream);
    }
    if (elem == INFER_ELEM_F32) {
        DeltaArgs<float> a;
        rc = make_args(a, proj, proj_stride, beta_off, decay, decay_stride, gate, gate_stride, conv, a_log, dt_bias, norm, ring, state,
                       num_slots, heads, kv_heads, dim, vdim, taps, eps, out, out_stride);
        return rc ? rc : launch_chunks(a, (const PortionDesc*)portions, num_portions, (const ChunkDesc*)chunks, num_chunks, records, o,
                                       row0, rows, ring_slot, positions, (hipStream_t)stream);
    }
    return INFER_KV_EUNSUPPORTED;
}
