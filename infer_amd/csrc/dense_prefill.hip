// Causal attention of long prompt portions over dense keys and values, for gfx950 (MI355X).  bf16 in, float32
// accumulate, output gate and softmax sink in the epilogue.  A key has two parts, either of which may be absent: one
// that the heads of a group share (latent attention: W_uk c, a group of one; grouped attention: the whole key), and
// one that all heads share (latent attention: the rotated part).  A query may see only the keys of its chunk or of a window
// (masks.h): a workgroup walks the keys that one of its queries sees.
//
// A wavefront owns 32 queries (two MFMA column tiles) of one head, a workgroup four wavefronts = 128
// consecutive queries, and walks the visible keys in steps of 32 that all four share through LDS (two
// buffers; the rows of the next two steps travel through registers meanwhile):
//   S^T[key, query] = [k_plain | k_rot][key, :] . q^T      KS k-steps of 32
//   O^T[v, query]  += V^T[v, key] . P^T                    VT row tiles of 16
// Row r of the score tile t is key 8 (r / 4) + 4 t + r % 4, so that a lane's eight scores are the eight
// consecutive keys the second product wants from it and P never leaves its registers.
// Two maps (two attentions over the same values, the output is their difference, normed): a wavefront owns 16 queries, and its
// two column tiles are their two maps, each against its own key.
#include "elem.h"
#include "masks.h"

namespace {

typedef short i16x4 __attribute__((ext_vector_type(4)));
typedef short i16x8 __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) i16x4 lds_i16x4;

constexpr int kStep = 32;
constexpr int kWaves = 4;
constexpr float kNoMax = 1e30f;         // minus the running maximum before a key was seen; finite, since a masked score is -inf
constexpr float kLazy = 8.f;            // log2 units a row's maximum may grow before the accumulators are rescaled

struct DensePrefillArgs {
    const __bf16* q; int64_t q_stride;        // [token][head * (dim + rot)]
    const __bf16* kp; int64_t kp_stride; int kp_head;   // [key][group of heads][dim]
    const __bf16* kr; int64_t kr_stride;      // [key][rot]
    const __bf16* v; int64_t v_stride; int v_head;      // [key][group of heads][vdim]
    const __bf16* gate; int64_t gate_stride;  // [token][head]
    const float* sink;                        // [head] or nullptr
    int group;                                // heads that share keys and values
    __bf16* out; int64_t out_stride;          // [token][head * vdim]
    const int32_t* cu_q;                      // first token row of each sequence (rows of q, gate, out)
    const int32_t* cu_k;                      // first key row of each
    int heads, dim, rot, vdim, nseq, qblocks;
    float scale_log2;
    KeyMask mask;
    bool biased;                              // scores lose distance_slope(head) per token of distance
    float out_scale;                          // of the output
    float lambda, eps;                        // two maps: rms(o1 - lambda o2) * out_scale
};

template <int KS, int VT, int MAPS>
__global__ void __launch_bounds__(64 * kWaves, 2) dense_prefill_kernel(DensePrefillArgs a) {
    constexpr int kTileQ = MAPS == 2 ? 0 : 16, kWaveQ = 32 / MAPS, kWgQ = kWaveQ * kWaves;   // queries: between the tiles, per wavefront, per workgroup
    constexpr int kKPitch = MAPS * KS * 64 + 16, kVPitch = VT * 32 + 16;              // bytes
    constexpr int kBuf = kStep * (kKPitch + kVPitch);
    constexpr int kNK = MAPS * KS * 4 * kStep / 256, kNV = (VT * 2 * kStep + 255) / 256;    // 16-byte chunks per thread
    __shared__ __attribute__((aligned(16))) unsigned char lds[2 * kBuf];
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int g = lane >> 4, n = lane & 15;
    // Workgroups go to the eight dies round-robin; die k works through the k-th contiguous eighth of the
    // (head, sequence, query block) space, so that the blocks that read the same keys share an L2.
    const unsigned total = gridDim.x, id = blockIdx.x;
    const unsigned die = id & 7u, per_die = total >> 3, extra = total & 7u;
    const unsigned wg = die * per_die + (die < extra ? die : extra) + (id >> 3);
    const int qblk = a.qblocks - 1 - (int)(wg % a.qblocks);      // late blocks see the most keys: first
    const int b = (int)((wg / a.qblocks) % a.nseq), h = (int)(wg / ((unsigned)a.qblocks * a.nseq));
    const int q_beg = a.cu_q[b], sq = a.cu_q[b + 1] - q_beg;
    const int k_beg = a.cu_k[b], sk = a.cu_k[b + 1] - k_beg;
    const int wq0 = qblk * kWgQ;
    if (wq0 >= sq) return;
    const int q0 = wq0 + kWaveQ * wave;
    const bool live = q0 < sq;
    const int shift = sk - sq;                                   // query i sees keys 0 .. i + shift
    const int last_q = wq0 + kWgQ < sq ? wq0 + kWgQ - 1 : sq - 1;
    const int nsteps = (last_q + shift + 1 + kStep - 1) / kStep;
    const int my_last = q0 + kWaveQ - 1 < sq ? q0 + kWaveQ - 1 : sq - 1;
    const int first_step = a.mask.first(wq0 + shift) / kStep, my_first = a.mask.first(q0 + shift) / kStep;
    const int my_steps = live ? (my_last + shift + 1 + kStep - 1) / kStep : 0;

    const int qk = a.dim + a.rot;
    bf16x8_t qreg[2][KS];
    int limit[2], lowest[2];
    const float slope = a.biased ? distance_slope(h, a.heads) * kLog2e / a.scale_log2 : 0.f;
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        const int qi = q0 + kTileQ * u + n;
        limit[u] = qi + shift;
        lowest[u] = a.mask.first(limit[u]);
        const __bf16* qp = a.q + (int64_t)(q_beg + (qi < sq ? qi : sq - 1)) * a.q_stride + (int64_t)(MAPS == 2 ? 2 * h + u : h) * qk + 8 * g;
#pragma unroll
        for (int j = 0; j < KS; ++j) {
            qreg[u][j] = bf16x8_t{};
            if (32 * j + 8 * g < qk) qreg[u][j] = *reinterpret_cast<const bf16x8_t*>(qp + 32 * j);
        }
    }

    // the columns behind the real sizes stay zero in both buffers
    for (int i = tid; i < 2 * kBuf / 16; i += 256) reinterpret_cast<u32x4_t*>(lds)[i] = u32x4_t{0u, 0u, 0u, 0u};

    // chunk i of this thread of the K and of the V tile: key, place, and a running pointer to its source
    const int hk = h / a.group;
    const int kc = qk / 8, vc = a.vdim / 8, dc = a.dim / 8;
    constexpr int kN = kNK + kNV;
    int c_key[kN], c_lds[kN], c_str[kN];                         // c_str: elements from one key to the next (checked below 2^24)
    const __bf16* c_src[kN];
#pragma unroll
    for (int i = 0; i < kN; ++i) {
        const bool is_k = i < kNK;
        const int c = tid + 256 * (is_k ? i : i - kNK), per = is_k ? MAPS * kc : vc;
        const int key = c / per, col = c - key * per;
        c_key[i] = key < kStep ? key : -1;                       // -1: no such chunk; it re-reads the first value and is not stored
        const int map = MAPS == 2 && col >= kc;
        c_lds[i] = is_k ? key * kKPitch + map * (KS * 64) + (col - map * kc) * 16 : kStep * kKPitch + key * kVPitch + col * 16;
        const bool rot = MAPS == 1 && is_k && col >= dc;
        c_str[i] = key >= kStep ? 0 : (int)(!is_k ? a.v_stride : rot ? a.kr_stride : a.kp_stride);
        const __bf16* base = !is_k ? a.v + (int64_t)hk * a.v_head + 8 * col
                             : rot ? a.kr + 8 * (col - dc) : a.kp + (int64_t)hk * a.kp_head + 8 * col;
        c_src[i] = (key < kStep ? base : a.v) + (int64_t)(k_beg + first_step * kStep + key) * c_str[i];
    }
    // Two steps are under way in registers while a third is consumed from LDS: a step is shorter than the
    // round trip to the second-level cache.
    u32x4_t st0[kN], st1[kN];
    auto fetch = [&](int s, u32x4_t (&st)[kN]) {
        const int over = kStep - (sk - s * kStep);               // keys behind the last one re-read it; their weights are zero
#pragma unroll
        for (int i = 0; i < kN; ++i) {
            const __bf16* p = c_src[i];
            if (over > 0) {
                const int key = c_key[i] > 0 ? c_key[i] : 0, last = kStep - 1 - over;
                if (key > last) p -= (int64_t)(key - last) * c_str[i];
            }
            st[i] = *reinterpret_cast<const u32x4_t*>(p);
            c_src[i] += (int64_t)kStep * c_str[i];
        }
    };
    auto put = [&](unsigned char* buf, const u32x4_t (&st)[kN]) {
#pragma unroll
        for (int i = 0; i < kN; ++i)
            if (c_key[i] >= 0) *reinterpret_cast<u32x4_t*>(buf + c_lds[i]) = st[i];
    };

    f32x4_t acc[2][VT], lacc[2];
    float m_neg[2];
    bf16x8_t ones;
#pragma unroll
    for (int i = 0; i < 8; ++i) ones[i] = (__bf16)1.f;
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        m_neg[u] = kNoMax;
        lacc[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < VT; ++t) acc[u][t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    }

    fetch(first_step, st0);
    if (nsteps > first_step + 1) fetch(first_step + 1, st1);
    __syncthreads();          // the zero fill
    put(lds, st0);
    __syncthreads();
    const int k_addr = (8 * (n >> 2) + (n & 3)) * kKPitch + 16 * g;
    const int v_addr = kStep * kKPitch + (8 * g + (n >> 2)) * kVPitch + (n & 3) * 8;
    // step s consumes buffer s % 2, requests step s + 2 into `ahead` and stores step s + 1, which is in `next`
    auto step = [&](int s, const unsigned char* buf, unsigned char* other, u32x4_t (&ahead)[kN], u32x4_t (&next)[kN]) {
        if (s + 2 < nsteps) fetch(s + 2, ahead);
        if (s >= my_first && s < my_steps) {
            const int tok0 = s * kStep;
            f32x4_t sc[2][2];
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                // the accumulators start at the bias of the distance
                const float from = MAPS == 1 && a.biased ? slope * (float)(tok0 + 8 * g - limit[u]) : 0.f;
#pragma unroll
                for (int t = 0; t < 2; ++t)
#pragma unroll
                    for (int e = 0; e < 4; ++e) sc[u][t][e] = MAPS == 1 ? from + slope * (float)(4 * t + e) : 0.f;
            }
#pragma unroll
            for (int j = 0; j < KS; ++j)
#pragma unroll
                for (int t = 0; t < 2; ++t) {
                    bf16x8_t kf = *reinterpret_cast<const bf16x8_t*>(buf + k_addr + 4 * t * kKPitch + 64 * j);
#pragma unroll
                    for (int u = 0; u < 2; ++u) {
                        if (MAPS == 2 && u == 1) kf = *reinterpret_cast<const bf16x8_t*>(buf + k_addr + 4 * t * kKPitch + 64 * (KS + j));
                        sc[u][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qreg[u][j], sc[u][t], 0, 0, 0);
                    }
                }
            bf16x8_t pb[2];
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                float sv[8];
#pragma unroll
                for (int t = 0; t < 2; ++t)
#pragma unroll
                    for (int e = 0; e < 4; ++e) sv[4 * t + e] = sc[u][t][e];
                if (tok0 + kStep - 1 > q0 + kTileQ * u + shift) {      // the earliest query of the tile does not see all of it
                    const int rel = limit[u] - tok0 - 8 * g;
#pragma unroll
                    for (int i = 0; i < 8; ++i)
                        if (i > rel) sv[i] = -INFINITY;
                }
                if (tok0 < a.mask.first(q0 + kTileQ * u + 15 + shift)) {   // nor the latest one
                    const int rel = lowest[u] - tok0 - 8 * g;
#pragma unroll
                    for (int i = 0; i < 8; ++i)
                        if (i < rel) sv[i] = -INFINITY;
                }
                float mx = sv[0];
#pragma unroll
                for (int i = 1; i < 8; ++i) mx = fmaxf(mx, sv[i]);
                mx = max_xor16_32(mx) * a.scale_log2;
                const bool grow = mx + m_neg[u] > kLazy;               // always with the first key that is seen
                if (__any(grow)) {
                    const float alpha = grow ? __builtin_amdgcn_exp2f(-m_neg[u] - mx) : 1.f;
                    m_neg[u] = grow ? -mx : m_neg[u];
                    lacc[u] *= alpha;
#pragma unroll
                    for (int t = 0; t < VT; ++t) acc[u][t] *= alpha;
                }
#pragma unroll
                for (int i = 0; i < 8; ++i) pb[u][i] = (__bf16)__builtin_amdgcn_exp2f(__builtin_fmaf(sv[i], a.scale_log2, m_neg[u]));
                lacc[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, pb[u], lacc[u], 0, 0, 0);
            }
#pragma unroll
            for (int t = 0; t < VT; ++t) {
                const i16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(buf + v_addr + 32 * t));
                const i16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_i16x4*)(buf + v_addr + 32 * t + 4 * kVPitch));
                const bf16x8_t vt = __builtin_bit_cast(bf16x8_t, (i16x8)__builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
#pragma unroll
                for (int u = 0; u < 2; ++u) acc[u][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, pb[u], acc[u][t], 0, 0, 0);
            }
        }
        if (s + 1 < nsteps) put(other, next);
        __syncthreads();
    };
    for (int s = first_step; s < nsteps; s += 2) {
        step(s, lds, lds + kBuf, st0, st1);
        if (s + 1 < nsteps) step(s + 1, lds + kBuf, lds, st1, st0);
    }
    if (!live) return;
    auto store = [&](int qi, auto value) {
        __bf16* o = a.out + (int64_t)(q_beg + qi) * a.out_stride + (int64_t)h * a.vdim + 4 * g;
#pragma unroll
        for (int t = 0; t < VT; ++t)
            if (16 * t + 4 * g < a.vdim) {
                bf16x4_t v;
#pragma unroll
                for (int e = 0; e < 4; ++e) v[e] = (__bf16)value(t, e);
                *reinterpret_cast<bf16x4_t*>(o + 16 * t) = v;
            }
    };
    auto gate_of = [&](int qi) { return a.gate ? sigmoid_f((float)a.gate[(int64_t)(q_beg + qi) * a.gate_stride + h]) : 1.f; };
    if constexpr (MAPS == 2) {
        const float f0 = lacc[0][0] > 0.f ? 1.f / lacc[0][0] : 0.f, f1 = lacc[1][0] > 0.f ? -a.lambda / lacc[1][0] : 0.f;
        float ss = 0.f;                                          // values behind the real size are zero
#pragma unroll
        for (int t = 0; t < VT; ++t)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                acc[0][t][e] = acc[0][t][e] * f0 + acc[1][t][e] * f1;
                ss += acc[0][t][e] * acc[0][t][e];
            }
        ss += __shfl_xor(ss, 16, 64);
        ss += __shfl_xor(ss, 32, 64);
        const int qi = q0 + n;
        if (qi >= sq) return;
        const float f = rsqrtf(ss / (float)a.vdim + a.eps) * a.out_scale * gate_of(qi);
        store(qi, [&](int t, int e) { return acc[0][t][e] * f; });
    } else {
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int qi = q0 + 16 * u + n;
            if (qi >= sq) continue;
            float l = lacc[u][0];
            if (a.sink && l > 0.f) l += __builtin_amdgcn_exp2f(a.sink[h] * kLog2e + m_neg[u]);
            const float f = (l > 0.f ? a.out_scale / l : 0.f) * gate_of(qi);
            store(qi, [&](int t, int e) { return acc[u][t][e] * f; });
        }
    }
}

// (k-steps, value tiles) the kernel is built for, smallest first
template <int KS, int VT, int MAPS = 1>
int go(const DensePrefillArgs& a, unsigned grid, hipStream_t st) {
    hipLaunchKernelGGL((dense_prefill_kernel<KS, VT, MAPS>), dim3(grid), dim3(64 * kWaves), 0, st, a);
    return (int)hipGetLastError();
}

// the checks that both forms of the entry share, and the launch
int run(DensePrefillArgs& a, int64_t num_seqs, int64_t max_seqlen_q, float scale, void* stream, int maps = 1) {
    if (num_seqs < 0 || max_seqlen_q < 0) return INFER_KV_EINVAL;
    if (num_seqs == 0 || max_seqlen_q == 0) return INFER_KV_OK;
    if (!a.q || !a.kp || !a.v || !a.out || !a.cu_q || !a.cu_k || !(scale > 0.f)) return INFER_KV_EINVAL;
    const int64_t qk = a.dim + a.rot;
    if (a.q_stride < a.heads * maps * qk || (a.gate && a.gate_stride < a.heads) || a.out_stride < (int64_t)a.heads * a.vdim) return INFER_KV_EINVAL;
    if (a.kp_stride >= (1 << 24) || a.kr_stride >= (1 << 24) || a.v_stride >= (1 << 24)) return INFER_KV_EINVAL;
    if (a.q_stride % 8 || a.kp_stride % 8 || a.kr_stride % 8 || a.v_stride % 8 || a.kp_head % 8 || a.v_head % 8 || a.out_stride % 4 ||
        !ptr_aligned(a.q, 16) || !ptr_aligned(a.kp, 16) || !ptr_aligned(a.kr, 16) || !ptr_aligned(a.v, 16) || !ptr_aligned(a.out, 8))
        return INFER_KV_EALIGN;
    const int64_t per_wg = 32 / maps * kWaves, qblocks = (max_seqlen_q + per_wg - 1) / per_wg, total = qblocks * num_seqs * a.heads;
    if (total > 0x7fffffff) return INFER_KV_EINVAL;
    a.nseq = (int)num_seqs;
    a.qblocks = (int)qblocks;
    a.scale_log2 = scale * kLog2e;
    hipStream_t st = (hipStream_t)stream;
    const unsigned grid = (unsigned)total;
    if (maps == 2) {
        if (qk <= 64 && a.vdim <= 64) return go<2, 4, 2>(a, grid, st);
        if (qk <= 64) return go<2, 8, 2>(a, grid, st);
        return go<4, 8, 2>(a, grid, st);
    }
    if (qk <= 64 && a.vdim <= 64) return go<2, 4>(a, grid, st);
    if (qk <= 128 && a.vdim <= 64) return go<4, 4>(a, grid, st);
    if (qk <= 128) return go<4, 8>(a, grid, st);
    if (qk <= 192) return go<6, 8>(a, grid, st);
    return go<8, 8>(a, grid, st);
}

bool served(int64_t dim, int64_t rot, int64_t vdim) {
    if (dim <= 0 || rot < 0 || vdim <= 0 || dim % 8 || rot % 8 || vdim % 8) return false;
    return dim + rot <= 256 && vdim <= 128;
}

}  // namespace

// 1 if the sizes are served by the kernel
extern "C" int infer_latent_prefill_supported(int64_t dim, int64_t rot, int64_t vdim) { return rot > 0 && served(dim, rot, vdim); }
extern "C" int infer_grouped_prefill_supported(int64_t dim, int64_t vdim) { return served(dim, 0, vdim); }

extern "C" int infer_latent_prefill(const void* q, int64_t q_stride, const void* kp, int64_t kp_stride, const void* kr,
                                    int64_t kr_stride, const void* v, int64_t v_stride, const void* gate, int64_t gate_stride,
                                    void* out, int64_t out_stride, const int32_t* cu_q, const int32_t* cu_k, int64_t num_seqs,
                                    int64_t max_seqlen_q, int64_t heads, int64_t dim, int64_t rot, int64_t vdim, float scale,
                                    void* stream) {
    if (heads < 1 || heads > 4096 || !infer_latent_prefill_supported(dim, rot, vdim)) return INFER_KV_EUNSUPPORTED;
    if (!kr || kp_stride < heads * dim || kr_stride < rot || v_stride < heads * vdim) return INFER_KV_EINVAL;
    DensePrefillArgs a{(const __bf16*)q, q_stride, (const __bf16*)kp, kp_stride, (int)dim, (const __bf16*)kr, kr_stride, (const __bf16*)v,
                       v_stride, (int)vdim, (const __bf16*)gate, gate_stride, nullptr, 1, (__bf16*)out, out_stride, cu_q, cu_k, (int)heads,
                       (int)dim, (int)rot, (int)vdim, 0, 0, 0.f, KeyMask{}, false, 1.f, 0.f, 0.f};
    if (!gate) return INFER_KV_EINVAL;
    return run(a, num_seqs, max_seqlen_q, scale, stream);
}

extern "C" int infer_grouped_prefill(const void* q, int64_t q_stride, const void* k, int64_t k_stride, int64_t k_head, const void* v,
                                     int64_t v_stride, int64_t v_head, const float* sink, const void* gate, int64_t gate_stride,
                                     void* out, int64_t out_stride, const int32_t* cu_q, const int32_t* cu_k, int64_t num_seqs,
                                     int64_t max_seqlen_q, int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim, float scale,
                                     void* stream) {
    if (heads < 1 || heads > 4096 || !infer_grouped_prefill_supported(dim, vdim)) return INFER_KV_EUNSUPPORTED;
    if (kv_heads < 1 || heads % kv_heads || k_head < 0 || v_head < 0 || k_stride < (kv_heads - 1) * k_head + dim ||
        v_stride < (kv_heads - 1) * v_head + vdim)
        return INFER_KV_EINVAL;
    DensePrefillArgs a{(const __bf16*)q, q_stride, (const __bf16*)k, k_stride, (int)k_head, nullptr, 0, (const __bf16*)v, v_stride,
                       (int)v_head, (const __bf16*)gate, gate_stride, sink, (int)(heads / kv_heads), (__bf16*)out, out_stride, cu_q, cu_k,
                       (int)heads, (int)dim, 0, (int)vdim, 0, 0, 0.f, KeyMask{}, false, 1.f, 0.f, 0.f};
    if (!gate) return INFER_KV_EINVAL;
    return run(a, num_seqs, max_seqlen_q, scale, stream);
}

// 1 if the sizes are served by the kernel
extern "C" int infer_masked_prefill_supported(int64_t maps, int64_t dim, int64_t vdim) {
    return maps >= 1 && maps <= 2 && served(dim, 0, vdim) && (maps == 1 || dim <= 128);
}

extern "C" int infer_masked_prefill(const void* q, int64_t q_stride, const void* k, int64_t k_stride, int64_t k_head, const void* v,
                                    int64_t v_stride, int64_t v_head, const float* sink, const void* gate, int64_t gate_stride,
                                    void* out, int64_t out_stride, const int32_t* cu_q, const int32_t* cu_k, int64_t num_seqs,
                                    int64_t max_seqlen_q, int64_t heads, int64_t kv_heads, int64_t maps, int64_t dim, int64_t vdim,
                                    float scale, int mask_kind, int64_t mask_size, int biased, float out_scale, float lambda, float eps,
                                    void* stream) {
    if (heads < 1 || heads > 4096 || !infer_masked_prefill_supported(maps, dim, vdim)) return INFER_KV_EUNSUPPORTED;
    if (kv_heads < 1 || heads % kv_heads || k_head < 0 || v_head < 0 || k_stride < (kv_heads - 1) * k_head + maps * dim ||
        v_stride < (kv_heads - 1) * v_head + vdim || (maps == 2 && (sink || biased)) || !mask_valid(mask_kind, mask_size))
        return INFER_KV_EINVAL;
    DensePrefillArgs a{(const __bf16*)q, q_stride, (const __bf16*)k, k_stride, (int)k_head, nullptr, 0, (const __bf16*)v, v_stride,
                       (int)v_head, (const __bf16*)gate, gate_stride, sink, (int)(heads / kv_heads), (__bf16*)out, out_stride, cu_q, cu_k,
                       (int)heads, (int)dim, 0, (int)vdim, 0, 0, 0.f, KeyMask{mask_kind, (int)mask_size}, biased != 0, out_scale, lambda, eps};
    return run(a, num_seqs, max_seqlen_q, scale, stream, (int)maps);
}
