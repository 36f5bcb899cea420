// Attention whose heads mix their softmax weights (talking_attention.hip), for long prompt portions, for gfx950 (MI355X).  bf16 in, float32
// accumulate; keys and values go straight from their pages (tile_pages.h) into operands.
//
//     w_h(i, j) = e^{s_h(i, j)} / (1 + sum_j' e^{s_h(i, j')}) ,   o_h(i) = c sum_j (sum_g T[h][g] w_g(i, j)) v_j
//
// A running rescale does not commute with the mixture, so denominators come first, and the scores are computed twice instead of passing
// through memory:
//   talk_lse_kernel   log2 of every (head, query)'s denominator; a wavefront owns 16 U queries of a head
//   talk_mix_kernel   a workgroup of eight wavefronts owns 16 QT queries and ALL heads, UH heads per wavefront, and walks the keys in
//                     steps of 32:
//       S^T[key, query] = K[key, :] . q^T           per wavefront its heads; weights e^{S - lse} go to LDS as two bf16 pieces each
//                                                   (2^-17), one record [head][piece] per (query, key)
//       P'^T[key, h]    = W^T[key, g] . T^T[g, h]    per wavefront 2 QT queries, the pieces side by side along k; to LDS as bf16
//       O^T[v, query]  += V^T[v, key] . P'^T[key, query]      per wavefront its heads
//                     Nothing is rescaled: what is added up is final, and the keys of a few queries can be split over workgroups, whose
//                     sums talk_sum_kernel adds up.  Between the barriers that enclose the mixture a wavefront computes the scores
//                     of the next step and the sums of this one, the two wavefronts of a vector unit in opposite order.
// A lane's eight results of the first two products are those of eight consecutive keys (tile_row_token).
#include <type_traits>

#include "elem.h"
#include "pieces.h"
#include "tile_pages.h"

namespace {

typedef uint32_t u32x2_t __attribute__((ext_vector_type(2)));

constexpr int kStep = kTileTokens;
constexpr int kLseWaves = 4;
constexpr int kMixWaves = 8;
constexpr float kLow = -1e30f;            // a maximum before any key was seen; finite, since hidden scores are -inf
constexpr float kLazy = 8.f;              // log2 units by which a sum's terms may exceed one before it is rescaled
constexpr float kBound = 100.f;           // log2 units: powers of scores below it add up in a float as they are

struct TalkPrefillArgs {
    const __bf16* q; int64_t q_stride;    // [token][head * dim]
    const __bf16* keys; const __bf16* values;                 // tile_pages.h
    int key_pad, vdim_pad;
    const int32_t* bt; int64_t bt_stride; int table_cols, block_size, num_blocks;
    const int32_t* seqs; const int32_t* cu_q; const int32_t* cu_k;
    int heads, kv_heads, dim, vdim, nseq, qblocks;
    float scale_log2;
    const __bf16* talk;                   // [heads][heads]
    float out_scale;
    __bf16* out; int64_t out_stride;      // [token][head * vdim]
    float* lse; int64_t tokens;           // [heads][tokens]
    int splits, split_steps;              // steps per split
    float* part;                          // [splits][tokens][heads * vdim], if splits > 1
};

// The tiles of 32 keys of a sequence, one behind the other; a tile lies in one block, whose id is looked up one block ahead.
struct PageWalk {
    typedef const __attribute__((address_space(4))) int32_t* Table;       // nobody writes it meanwhile: scalar loads
    Table bt;
    int tiles_per_block, col, in_block, id, next_id;
    __device__ __forceinline__ int lookup(const TalkPrefillArgs& a, int c) const {
        const int b = bt[c < a.table_cols ? c : a.table_cols - 1];
        return b < 0 ? 0 : (b >= a.num_blocks ? a.num_blocks - 1 : b);
    }
    __device__ __forceinline__ PageWalk(const TalkPrefillArgs& a, int seq, int first = 0) {
        bt = (Table)(uintptr_t)(a.bt + (int64_t)a.seqs[seq] * a.bt_stride);
        tiles_per_block = a.block_size / kStep;
        col = first / tiles_per_block;
        in_block = first - col * tiles_per_block;
        id = lookup(a, col);
        next_id = lookup(a, col + 1);
    }
    // the tile's number among the tiles of all blocks of one head (of kv_heads), for key/value head 0; then moves on
    __device__ __forceinline__ int64_t next(const TalkPrefillArgs& a) {
        const int64_t at = (int64_t)id * a.kv_heads * tiles_per_block + in_block;
        if (++in_block == tiles_per_block) {
            in_block = 0;
            ++col;
            id = next_id;
            next_id = lookup(a, col + 1);
        }
        return at;
    }
};

// Workgroups go to the eight dies round-robin.  A die works on its own share of `pairs`, on the late query blocks, which see the most
// keys, first.  False: no such pair.
__device__ __forceinline__ bool place_of_block(unsigned id, int pairs, int qblocks, int& pair, int& qblk) {
    const int die = (int)(id & 7u), i = (int)(id >> 3), per_die = (pairs + 7) / 8;
    pair = die * per_die + i % per_die;
    qblk = qblocks - 1 - i / per_die;
    return pair < pairs;
}

// An operand at an address that all lanes share plus a byte offset of each
__device__ __forceinline__ bf16x8_t load_operand(const __bf16* base, unsigned lane_bytes) {
    return *reinterpret_cast<const bf16x8_t*>(reinterpret_cast<const char*>(base) + lane_bytes);
}

// BOUNDED: all scores are below kBound, so that their powers need no maximum.
template <int KS, int U, bool BOUNDED>
__global__ void __launch_bounds__(64 * kLseWaves, 2) talk_lse_kernel(TalkPrefillArgs a) {
    constexpr int kLseQ = 16 * U;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, n = lane & 15;
    int pair, qblk;
    if (!place_of_block(blockIdx.x, a.nseq * a.heads, a.qblocks, pair, qblk)) return;
    const int b = pair / a.heads, h = pair - b * a.heads;
    const int q_beg = a.cu_q[b], sq = a.cu_q[b + 1] - q_beg, sk = a.cu_k[b + 1] - a.cu_k[b], shift = sk - sq;
    const int q0 = (qblk * kLseWaves + wave) * kLseQ;
    if (q0 >= sq) return;
    const int last_q = q0 + kLseQ < sq ? q0 + kLseQ - 1 : sq - 1, steps = (last_q + shift) / kStep + 1;
    bf16x8_t q[U][KS];
    float m[U], l[U];
    int limit[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
        const int qi = q0 + 16 * u + n < sq ? q0 + 16 * u + n : sq - 1;
        limit[u] = qi + shift;
        m[u] = BOUNDED ? 0.f : kLow;
        l[u] = 0.f;
        const __bf16* qp = a.q + (int64_t)(q_beg + qi) * a.q_stride + (int64_t)h * a.dim + 8 * g;
#pragma unroll
        for (int j = 0; j < KS; ++j) {
            q[u][j] = bf16x8_t{};
            if (32 * j + 8 * g < a.dim) q[u][j] = *reinterpret_cast<const bf16x8_t*>(qp + 32 * j);
        }
    }
    int k_step[KS];                                   // k-steps behind the size repeat the first one, which meets zeros
#pragma unroll
    for (int j = 0; j < KS; ++j) k_step[j] = tile_key_entry(0, 32 * j < a.key_pad ? 32 * j : 0);
    const int64_t head_at = (int64_t)(h / (a.heads / a.kv_heads)) * a.block_size * a.key_pad;
    const unsigned k_lane = 2u * (unsigned)tile_key_entry(tile_row_token(n, 0), 8 * g);
    PageWalk walk(a, b);
    bf16x8_t kf[2][KS];
    auto fetch = [&]() {
        const __bf16* src = a.keys + walk.next(a) * kStep * a.key_pad + head_at;
#pragma unroll
        for (int x = 0; x < 2; ++x)
#pragma unroll
            for (int j = 0; j < KS; ++j) kf[x][j] = load_operand(src + k_step[j] + tile_key_entry(tile_row_token(0, x), 0), k_lane);
    };
    fetch();
    for (int s = 0; s < steps; ++s) {
        f32x4_t sc[U][2];
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int x = 0; x < 2; ++x) sc[u][x] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < KS; ++j)
#pragma unroll
            for (int x = 0; x < 2; ++x)
#pragma unroll
                for (int u = 0; u < U; ++u) sc[u][x] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[x][j], q[u][j], sc[u][x], 0, 0, 0);
        if (s + 1 < steps) fetch();
        const int tok0 = s * kStep;
#pragma unroll
        for (int u = 0; u < U; ++u) {
            float sv[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) sv[i] = sc[u][i >> 2][i & 3];
            if (tok0 + kStep - 1 > q0 + 16 * u + shift) {        // the earliest query of the tile does not see all of it
                const int rel = limit[u] - tok0 - 8 * g;
#pragma unroll
                for (int i = 0; i < 8; ++i)
                    if (i > rel) sv[i] = -INFINITY;
            }
            if constexpr (BOUNDED) {
#pragma unroll
                for (int i = 0; i < 8; ++i) l[u] += __builtin_amdgcn_exp2f(sv[i] * a.scale_log2);
            } else {
                float mx = sv[0];
#pragma unroll
                for (int i = 1; i < 8; ++i) mx = fmaxf(mx, sv[i]);
                mx *= a.scale_log2;
                const bool grow = mx > m[u] + kLazy;
                if (__any(grow)) {
                    l[u] *= grow ? __builtin_amdgcn_exp2f(m[u] - mx) : 1.f;
                    m[u] = grow ? mx : m[u];
                }
#pragma unroll
                for (int i = 0; i < 8; ++i) l[u] += __builtin_amdgcn_exp2f(__builtin_fmaf(sv[i], a.scale_log2, -m[u]));
            }
        }
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
#pragma unroll
        for (int x = 16; x <= 32; x *= 2) {
            const float m2 = __shfl_xor(m[u], x, 64), l2 = __shfl_xor(l[u], x, 64), top = fmaxf(m[u], m2);
            l[u] = l[u] * exp2f(m[u] - top) + l2 * exp2f(m2 - top);
            m[u] = top;
        }
        const float top = fmaxf(m[u], 0.f);
        if (g == 0 && q0 + 16 * u + n < sq)
            a.lse[(int64_t)h * a.tokens + q_beg + q0 + 16 * u + n] = top + log2f(l[u] * exp2f(m[u] - top) + exp2f(-top));
    }
}

// Address in LDS of byte `at` of the record of (query q, key token), REC bytes long.  Lanes that write (16 queries, one key) and lanes
// that read (16 keys of tile_row_token, one query) meet all banks.  For the second eight of 16 queries the halves of every 16 bytes
// are swapped (`swapped`).  What a query, a key and `at` contribute is independent.
template <int REC>
__device__ __forceinline__ int record_place(int q, int token, int at) {
    const int low = REC == 128 ? (token & 3) | (token >> 1 & 4) : REC == 64 ? (token >> 1 & 1) | (token >> 2 & 2) : token >> 3 & 1;
    return (q * kStep + token) * REC + at ^ (low << 4) ^ ((q & 15) << 4) ^ (q & 8);
}
__device__ __forceinline__ bool swapped(int q) { return q & 8; }
template <int HP>
__device__ __forceinline__ int mixed_place(int q, int slot, int g) { return (q * HP + (slot ^ (q & (HP - 1)))) * 64 + 16 * (g ^ ((q >> 2) & 3)); }

// A value that the compiler takes for a new one: what is computed from it is not kept in registers over the whole loop.
__device__ __forceinline__ int renewed(int x) {
    asm volatile("" : "+v"(x));
    return x;
}

// SHARE: the heads of a wavefront have one key/value head.
template <int KS, int VT, int UH, int QT, bool SHARE>
__global__ void __launch_bounds__(64 * kMixWaves) __attribute__((amdgpu_waves_per_eu(2, 2))) talk_mix_kernel(TalkPrefillArgs a) {
    constexpr int HP = kMixWaves * UH, Q = 16 * QT;              // head slots, queries
    constexpr int kRec = 4 * HP;                                 // bytes of a record: every head's weight in two pieces
    constexpr int KP = UH == 4 ? 2 : 1, RT = UH == 4 ? 2 : 1;    // k-steps and head tiles of the mixture
    constexpr int UK = SHARE ? 1 : UH, UW = UH / UK;             // key heads of a wavefront, query heads of each
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];
    unsigned char* wbuf = lds;                                   // [Q][32 keys][kRec]
    unsigned char* pbuf = wbuf + Q * kStep * kRec;               // [Q][HP][32 keys] bf16
    bf16x8_t* talk = reinterpret_cast<bf16x8_t*>(pbuf + Q * HP * 2 * kStep);       // [2][KP][RT][64]
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), g = lane >> 4, n = lane & 15;
    int b, qblk;
    const int split = blockIdx.y;
    if (a.nseq % 8 == 0) {                                       // a sequence belongs to one die, whose second-level cache has its keys
        if (!place_of_block(blockIdx.x, a.nseq, a.qblocks, b, qblk)) return;
    } else {
        b = (int)(blockIdx.x % (unsigned)a.nseq);
        qblk = a.qblocks - 1 - (int)(blockIdx.x / (unsigned)a.nseq);
    }
    const int q_beg = a.cu_q[b], sq = a.cu_q[b + 1] - q_beg, sk = a.cu_k[b + 1] - a.cu_k[b], shift = sk - sq;
    const int q0 = qblk * Q;
    if (q0 >= sq) return;
    const int last_q = q0 + Q < sq ? q0 + Q - 1 : sq - 1, all_steps = (last_q + shift) / kStep + 1;
    const int s0 = split * a.split_steps, steps = s0 + a.split_steps < all_steps ? s0 + a.split_steps : all_steps;
    if (s0 >= steps) return;
    const int group = a.heads / a.kv_heads;

    bf16x8_t q[UH][QT][KS];
    float lse[UH][QT];
    int limit[QT];
    int64_t k_head[UK], v_head[UK];
#pragma unroll
    for (int u = 0; u < UH; ++u) {
        const int h = wave * UH + u < a.heads ? wave * UH + u : a.heads - 1;         // a surplus slot repeats the last head and meets zeros in T
        if (u % UW == 0) {
            k_head[u / UW] = (int64_t)(h / group) * a.block_size * a.key_pad;
            v_head[u / UW] = (int64_t)(h / group) * a.block_size * a.vdim_pad;
        }
#pragma unroll
        for (int t = 0; t < QT; ++t) {
            const int qi = q0 + 16 * t + n < sq ? q0 + 16 * t + n : sq - 1;
            limit[t] = qi + shift;
            lse[u][t] = a.lse[(int64_t)h * a.tokens + q_beg + qi];
            const __bf16* qp = a.q + (int64_t)(q_beg + qi) * a.q_stride + (int64_t)h * a.dim + 8 * g;
#pragma unroll
            for (int j = 0; j < KS; ++j) {
                q[u][t][j] = bf16x8_t{};
                if (32 * j + 8 * g < a.dim) q[u][t][j] = *reinterpret_cast<const bf16x8_t*>(qp + 32 * j);
            }
        }
    }
    // T^T: entry i of lane (g, n) is column (head) 16 s + 4 g + i / 2 of row (head) 16 r + n, once for either piece; behind it the same
    // for records whose halves are swapped
    for (int i = tid; i < 2 * KP * RT * 64; i += 64 * kMixWaves) {
        const int s = i / (64 * RT) % KP, r = i / 64 % RT, to = 16 * r + i % 16;
        bf16x8_t x;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const int from = 16 * s + 4 * (i % 64 / 16) + (i < KP * RT * 64 ? e : e ^ 4) / 2;
            x[e] = from < HP && from < a.heads && to < a.heads ? a.talk[(int64_t)to * a.heads + from] : (__bf16)0.f;
        }
        talk[i] = x;
    }

    f32x4_t acc[UH][QT][VT];
#pragma unroll
    for (int u = 0; u < UH; ++u)
#pragma unroll
        for (int t = 0; t < QT; ++t)
#pragma unroll
            for (int v = 0; v < VT; ++v) acc[u][t][v] = f32x4_t{0.f, 0.f, 0.f, 0.f};

    PageWalk walk(a, b, s0);
    const unsigned k_lane = 2u * (unsigned)tile_key_entry(tile_row_token(n, 0), 8 * g), v_lane = 2u * (unsigned)tile_value_entry(8 * g, n);
    bf16x8_t kf[KS];
    // half x of the keys of head uk; k-steps behind the size repeat the first one, which meets zeros in q
    auto fetch_k = [&](int64_t tile, int uk, int x) __attribute__((always_inline)) {
        const __bf16* src = a.keys + tile * kStep * a.key_pad + k_head[uk] + tile_key_entry(tile_row_token(0, x), 0);
#pragma unroll
        for (int j = 0; j < KS; ++j) kf[j] = load_operand(src + tile_key_entry(0, 32 * j < a.key_pad ? 32 * j : 0), k_lane);
    };
    constexpr int kRing = UH == 2 ? 3 : 4;                                     // value operands under way
    bf16x8_t vf[kRing];
    // operand i of the step: tile i % VT of head i / VT; tiles behind the size repeat the first one and are not stored
    auto fetch_v = [&](int64_t tile, int i) __attribute__((always_inline)) {
        const int v = i % VT;
        vf[i % kRing] = load_operand(a.values + tile * kStep * a.vdim_pad + v_head[i / VT] + tile_value_entry(0, 16 * v < a.vdim_pad ? 16 * v : 0), v_lane);
    };
    const int w_fixed = record_place<kRec>(n, 8 * g, wave * UH * 4);
    const int whole = (q0 + shift + 1) / kStep;                  // steps of which the first query sees every key

    // scores and weights of step s, half of the keys of a key head at a time; its first keys are in kf
    auto scores = [&](auto masked, int s, int64_t tile) __attribute__((always_inline)) {
        constexpr bool MASKED = decltype(masked)::value;
        const int tok0 = s * kStep, w_base = renewed(w_fixed);
#pragma unroll
        for (int i = 0; i < 2 * UK; ++i) {
            const int uk = i / 2, x = i % 2;
            // two score tiles at a time: of two heads, or of two query tiles
            constexpr int GW = UW >= 2 ? 2 : 1, GT = UW >= 2 || QT == 1 ? 1 : 2;
#pragma unroll
            for (int w0 = 0; w0 < UW; w0 += GW)
#pragma unroll
                for (int t0 = 0; t0 < QT; t0 += GT) {
                    f32x4_t sc[GW][GT];
#pragma unroll
                    for (int w = 0; w < GW; ++w)
#pragma unroll
                        for (int t = 0; t < GT; ++t) sc[w][t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                    for (int j = 0; j < KS; ++j)
#pragma unroll
                        for (int w = 0; w < GW; ++w)
#pragma unroll
                            for (int t = 0; t < GT; ++t)
                                sc[w][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[j], q[uk * UW + w0 + w][t0 + t][j], sc[w][t], 0, 0, 0);
                    if (w0 + GW == UW && t0 + GT == QT && i + 1 < 2 * UK) fetch_k(tile, (i + 1) / 2, (i + 1) % 2);   // these are used up
#pragma unroll
                    for (int t = 0; t < GT; ++t) {
                        uint32_t pieces[GW][4];
#pragma unroll
                        for (int w = 0; w < GW; ++w)
#pragma unroll
                            for (int e = 0; e < 4; ++e) {
                                float p = __builtin_amdgcn_exp2f(__builtin_fmaf(sc[w][t][e], a.scale_log2, -lse[uk * UW + w0 + w][t0 + t]));
                                if (MASKED && e > limit[t0 + t] - tok0 - 8 * g - 4 * x) p = 0.f;
                                pieces[w][e] = round_pack(head(p), p - head(p));
                            }
#pragma unroll
                        for (int e = 0; e < 4; ++e) {
                            unsigned char* to = wbuf + (w_base ^ record_place<kRec>(0, 4 * x + e, (uk * UW + w0) * 4)) + (t0 + t) * (16 * kStep * kRec);
                            if constexpr (GW == 2) *reinterpret_cast<u32x2_t*>(to) = u32x2_t{pieces[0][e], pieces[1][e]};
                            else *reinterpret_cast<uint32_t*>(to) = pieces[0][e];
                        }
                    }
                }
        }
    };
    // the mixture, for queries 2 QT wave and on
    auto mix = [&]() __attribute__((always_inline)) {
        const int g = renewed(lane >> 4), n = renewed(lane & 15);
        bf16x8_t tf[KP][RT];
#pragma unroll
        for (int y = 0; y < KP; ++y)
#pragma unroll
            for (int r = 0; r < RT; ++r) tf[y][r] = talk[((swapped(2 * QT * wave) ? KP : 0) + y) * RT * 64 + r * 64 + lane];
#pragma unroll
        for (int k = 0; k < 2 * QT; ++k) {
            if (UH == 4) __builtin_amdgcn_sched_barrier(0);      // one query at a time: registers
            const int qi = 2 * QT * wave + k;
            f32x4_t mixed[RT][2];
#pragma unroll
            for (int x = 0; x < 2; ++x) {
#pragma unroll
                for (int r = 0; r < RT; ++r) mixed[r][x] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int y = 0; y < KP; ++y) {
                    const bf16x8_t wf = *reinterpret_cast<const bf16x8_t*>(wbuf + record_place<kRec>(qi, tile_row_token(n, x), 64 * y + 16 * (UH == 1 ? g & 1 : g) ^ (qi & 8)));
#pragma unroll
                    for (int r = 0; r < RT; ++r) mixed[r][x] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf, tf[y][r], mixed[r][x], 0, 0, 0);
                }
            }
#pragma unroll
            for (int r = 0; r < RT; ++r) {
                bf16x8_t p;
#pragma unroll
                for (int i = 0; i < 8; ++i) p[i] = (__bf16)mixed[r][i >> 2][i & 3];
                const int to = 16 * r + n;
                if (HP >= 16 || to < HP) *reinterpret_cast<bf16x8_t*>(pbuf + mixed_place<HP>(qi, to, g)) = p;
            }
        }
    };
    // weighted sum of the values of step s, the first of which are in vf; behind it kf has the first keys of next_tile
    auto sums = [&](auto masked, int s, int64_t tile, int64_t next_tile) __attribute__((always_inline)) {
        constexpr bool MASKED = decltype(masked)::value;         // some values lie behind the last one
        const int left = sk - s * kStep;
        const int g = renewed(lane >> 4), n = renewed(lane & 15);
#pragma unroll
        for (int uk = 0; uk < UK; ++uk) {
            bf16x8_t pb[UW][QT];
#pragma unroll
            for (int w = 0; w < UW; ++w)
#pragma unroll
                for (int t = 0; t < QT; ++t) pb[w][t] = *reinterpret_cast<const bf16x8_t*>(pbuf + mixed_place<HP>(16 * t + n, wave * UH + uk * UW + w, g));
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                const int i = uk * VT + v;
                bf16x8_t x = vf[i % kRing];
                if constexpr (MASKED)                        // values behind the last one may be anything
#pragma unroll
                    for (int e = 0; e < 8; ++e)
                        if (8 * g + e >= left) x[e] = (__bf16)0.f;
#pragma unroll
                for (int w = 0; w < UW; ++w)
#pragma unroll
                    for (int t = 0; t < QT; ++t) acc[uk * UW + w][t][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, pb[w][t], acc[uk * UW + w][t][v], 0, 0, 0);
                if (i + kRing < UK * VT) fetch_v(tile, i + kRing);
                if (i + kRing == UK * VT) {                  // the next step's first keys take the place of the last values
                    __builtin_amdgcn_sched_barrier(0);
                    fetch_k(next_tile, 0, 0);
                }
            }
        }
    };
    auto first_values = [&](int64_t tile) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < kRing; ++i) fetch_v(tile, i);
    };
    // tiles of this step, the next one and the one behind it; behind the last one it is repeated
    int64_t tile = walk.next(a), tile1 = s0 + 1 < steps ? walk.next(a) : tile, tile2 = s0 + 2 < steps ? walk.next(a) : tile1;
    __syncthreads();                                             // T
    // A wavefront's part of the walk; both forms meet the same barriers.  Loops of their own, since accumulators that several branches
    // change would be copied where these meet.
    auto run = [&](auto first) __attribute__((always_inline)) {
        constexpr bool SUMS_FIRST = decltype(first)::value;
        fetch_k(tile, 0, 0);
        if (s0 < whole) scores(std::false_type{}, s0, tile);
        else scores(std::true_type{}, s0, tile);
        if constexpr (SUMS_FIRST) first_values(tile);
        else fetch_k(tile1, 0, 0);
        __syncthreads();
        auto step = [&](auto masked, int s) __attribute__((always_inline)) {
            mix();
            __syncthreads();
            if constexpr (SUMS_FIRST) {
                sums(masked, s, tile, tile1);
                if (!decltype(masked)::value || s + 1 < steps) scores(masked, s + 1, tile1);
                first_values(tile1);
            } else {
                if (!decltype(masked)::value || s + 1 < steps) scores(masked, s + 1, tile1);
                first_values(tile);
                sums(masked, s, tile, tile2);
            }
            __syncthreads();
            tile = tile1;
            tile1 = tile2;
            if (s + 3 < steps) tile2 = walk.next(a);
        };
        const int plain = whole < steps ? whole : steps;
        int s = s0;
        for (; s + 1 < plain; ++s) step(std::false_type{}, s);
        for (; s < steps; ++s) step(std::true_type{}, s);
    };
    if (wave < kMixWaves / 2) run(std::true_type{});
    else run(std::false_type{});
#pragma unroll
    for (int u = 0; u < UH; ++u) {
        const int h = wave * UH + u;
        if (h >= a.heads) continue;
#pragma unroll
        for (int t = 0; t < QT; ++t) {
            const int qi = q0 + 16 * t + n;
            if (qi >= sq) continue;
            __bf16* o = a.out + (int64_t)(q_beg + qi) * a.out_stride + (int64_t)h * a.vdim + 4 * g;
            float* part = a.part + (((int64_t)split * a.tokens + q_beg + qi) * a.heads + h) * a.vdim + 4 * g;
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                if (16 * v + 4 * g >= a.vdim) continue;
                if (a.splits > 1) {
                    *reinterpret_cast<f32x4_t*>(part + 16 * v) = acc[u][t][v];
                    continue;
                }
                bf16x4_t x;
#pragma unroll
                for (int e = 0; e < 4; ++e) x[e] = (__bf16)(acc[u][t][v][e] * a.out_scale);
                *reinterpret_cast<bf16x4_t*>(o + 16 * v) = x;
            }
        }
    }
}

// Sums of the splits.  Workgroup: 1024 columns of a token.  queries: of a workgroup of talk_mix_kernel.
__global__ void __launch_bounds__(256) talk_sum_kernel(TalkPrefillArgs a, int queries) {
    const int64_t c = ((int64_t)blockIdx.y * 256 + threadIdx.x) * 4, cols = (int64_t)a.heads * a.vdim;
    const int b = blockIdx.z, q_beg = a.cu_q[b], sq = a.cu_q[b + 1] - q_beg, sk = a.cu_k[b + 1] - a.cu_k[b], qi = blockIdx.x;
    if (qi >= sq || c >= cols) return;
    const int last = (qi / queries + 1) * queries, last_q = last < sq ? last - 1 : sq - 1, steps = (last_q + sk - sq) / kStep + 1;
    const float* p = a.part + (q_beg + qi) * cols + c;
    f32x4_t sum = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s * a.split_steps < steps; ++s) sum += *reinterpret_cast<const f32x4_t*>(p + s * a.tokens * cols);
    bf16x4_t x;
#pragma unroll
    for (int e = 0; e < 4; ++e) x[e] = (__bf16)(sum[e] * a.out_scale);
    *reinterpret_cast<bf16x4_t*>(a.out + (int64_t)(q_beg + qi) * a.out_stride + c) = x;
}

// workgroups of the mixture that are worth having: two for every compute unit, since some see more keys than others
constexpr int64_t kWorkgroups = 512;
// queries of a workgroup, in tiles of 16, and splits of the keys.  A split has at least eight steps.
void plan(int64_t heads, int64_t num_seqs, int64_t max_seqlen_q, int64_t max_keys, int& tiles, int& splits, int& split_steps) {
    auto groups = [&](int t) { return (max_seqlen_q + 16 * t - 1) / (16 * t) * num_seqs; };
    const int most = heads <= 8 ? 4 : heads <= 16 ? 2 : 1, least = heads <= 8 ? 2 : 1;
    tiles = groups(most) >= kWorkgroups ? most : least;
    const int64_t steps = (max_keys + kStep - 1) / kStep;
    int64_t n = kWorkgroups / (groups(tiles) > 0 ? groups(tiles) : 1);
    if (n > steps / 8) n = steps / 8;
    if (n > 8) n = 8;
    if (n < 1) n = 1;
    split_steps = (int)((steps + n - 1) / n);
    if (split_steps < 1) split_steps = 1;
    splits = (int)((steps + split_steps - 1) / split_steps);
    if (splits < 1) splits = 1;
}

template <int KS, int U>
int launch_lse_of(TalkPrefillArgs a, int64_t max_seqlen_q, bool bounded, hipStream_t st) {
    const int64_t per = 16 * U * kLseWaves, qblocks = (max_seqlen_q + per - 1) / per, total = ((int64_t)a.nseq * a.heads + 7) / 8 * 8 * qblocks;
    if (total > 0x7fffffff) return INFER_KV_EINVAL;
    a.qblocks = (int)qblocks;
    if (bounded) hipLaunchKernelGGL((talk_lse_kernel<KS, U, true>), dim3((unsigned)total), dim3(64 * kLseWaves), 0, st, a);
    else hipLaunchKernelGGL((talk_lse_kernel<KS, U, false>), dim3((unsigned)total), dim3(64 * kLseWaves), 0, st, a);
    return (int)hipGetLastError();
}
template <int KS>
int launch_lse(const TalkPrefillArgs& a, int64_t max_seqlen_q, bool bounded, hipStream_t st) {
    // few queries: more wavefronts with fewer of them each
    if ((max_seqlen_q + 63) / 64 * a.nseq * a.heads < 2048) return launch_lse_of<KS, 2>(a, max_seqlen_q, bounded, st);
    return launch_lse_of<KS, 4>(a, max_seqlen_q, bounded, st);
}

template <int KS, int VT, int UH, int QT, bool SHARE>
int launch_mix(TalkPrefillArgs a, int64_t max_seqlen_q, hipStream_t st) {
    const int64_t qblocks = (max_seqlen_q + 16 * QT - 1) / (16 * QT), total = qblocks * a.nseq;
    if (total > 0x7fffffff) return INFER_KV_EINVAL;
    a.qblocks = (int)qblocks;
    auto kernel = &talk_mix_kernel<KS, VT, UH, QT, SHARE>;
    constexpr size_t lds = (size_t)16 * QT * kStep * kMixWaves * UH * (4 + 2) + (UH == 4 ? 4 : 1) * 2048;
    static_assert(lds <= 160 * 1024, "LDS of a compute unit");
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return (int)e;
    hipLaunchKernelGGL(kernel, dim3((unsigned)total, (unsigned)a.splits), dim3(64 * kMixWaves), lds, st, a);
    if (a.splits > 1) {
        const unsigned columns = (unsigned)(((int64_t)a.heads * a.vdim + 1023) / 1024);
        hipLaunchKernelGGL(talk_sum_kernel, dim3((unsigned)max_seqlen_q, columns, (unsigned)a.nseq), dim3(256), 0, st, a, 16 * QT);
    }
    return (int)hipGetLastError();
}

template <int KS, int VT>
int launch(const TalkPrefillArgs& a, int64_t max_seqlen_q, bool bounded, int tiles, hipStream_t st) {
    const int rc = launch_lse<KS>(a, max_seqlen_q, bounded, st);
    if (rc) return rc;
    const int group = a.heads / a.kv_heads;
    if (a.heads <= 8) return tiles == 4 ? launch_mix<KS, VT, 1, 4, true>(a, max_seqlen_q, st) : launch_mix<KS, VT, 1, 2, true>(a, max_seqlen_q, st);
    if (a.heads <= 16 && group % 2 == 0)
        return tiles == 2 ? launch_mix<KS, VT, 2, 2, true>(a, max_seqlen_q, st) : launch_mix<KS, VT, 2, 1, true>(a, max_seqlen_q, st);
    if (a.heads <= 16) return tiles == 2 ? launch_mix<KS, VT, 2, 2, false>(a, max_seqlen_q, st) : launch_mix<KS, VT, 2, 1, false>(a, max_seqlen_q, st);
    return group % 4 == 0 ? launch_mix<KS, VT, 4, 1, true>(a, max_seqlen_q, st) : launch_mix<KS, VT, 4, 1, false>(a, max_seqlen_q, st);
}

}  // namespace

// 1 if the sizes are served
extern "C" int infer_talking_prefill_supported(int64_t heads, int64_t dim, int64_t vdim) {
    return heads >= 1 && heads <= 32 && dim >= 8 && dim <= 128 && dim % 8 == 0 && vdim >= 8 && vdim <= 128 && vdim % 8 == 0;
}

extern "C" int64_t infer_talking_prefill_workspace_floats(int64_t heads, int64_t vdim, int64_t num_seqs, int64_t tokens, int64_t max_seqlen_q,
                                                          int64_t max_keys) {
    if (heads < 1 || vdim < 1 || num_seqs < 1 || tokens < 1 || max_seqlen_q < 1 || max_keys < 1) return 0;
    int tiles, splits, split_steps;
    plan(heads, num_seqs, max_seqlen_q, max_keys, tiles, splits, split_steps);
    const int64_t lse = (heads * tokens + 3) / 4 * 4;
    return lse + (splits > 1 ? splits * tokens * heads * vdim : 0);
}

extern "C" int infer_talking_prefill(const void* q, int64_t q_stride, const void* keys, const void* values, int64_t key_pad,
                                     int64_t vdim_pad, const int32_t* block_table, int64_t bt_stride, int64_t table_cols,
                                     int64_t block_size, int64_t num_blocks, const int32_t* seqs, const int32_t* cu_q,
                                     const int32_t* cu_k, int64_t num_seqs, int64_t tokens, int64_t max_seqlen_q,
                                     int64_t max_keys, int64_t heads,
                                     int64_t kv_heads, int64_t dim, int64_t vdim, float scale, const void* talk, float out_scale,
                                     float max_score, void* out, int64_t out_stride, float* workspace, int64_t workspace_floats, void* stream) {
    if (!infer_talking_prefill_supported(heads, dim, vdim)) return INFER_KV_EUNSUPPORTED;
    if (num_seqs < 0 || max_seqlen_q < 0 || tokens < 0 || max_seqlen_q > 0x7fffffff || max_seqlen_q > tokens || max_keys < max_seqlen_q ||
        max_keys > 0x7fffffe0 || num_seqs > 65535)
        return INFER_KV_EINVAL;
    if (num_seqs == 0 || max_seqlen_q == 0) return INFER_KV_OK;
    if (!q || !keys || !values || !block_table || !seqs || !cu_q || !cu_k || !talk || !out || kv_heads < 1 || heads % kv_heads ||
        q_stride < heads * dim || out_stride < heads * vdim || key_pad != (dim + 31) / 32 * 32 || vdim_pad != (vdim + 31) / 32 * 32 ||
        block_size < kStep || block_size % kStep || block_size > (1 << 20) || table_cols < 1 || table_cols * block_size > 0x7fffffff || bt_stride < table_cols || num_blocks < 1 ||
        num_blocks > 0x7fffffff || !(scale > 0.f))
        return INFER_KV_EINVAL;
    if (q_stride % 8 || out_stride % 4 || !ptr_aligned(q, 16) || !ptr_aligned(keys, 16) || !ptr_aligned(values, 16) || !ptr_aligned(out, 8))
        return INFER_KV_EALIGN;
    if (!workspace || !ptr_aligned(workspace, 16) ||
        workspace_floats < infer_talking_prefill_workspace_floats(heads, vdim, num_seqs, tokens, max_seqlen_q, max_keys))
        return INFER_KV_EWORKSPACE;
    int tiles, splits, split_steps;
    plan(heads, num_seqs, max_seqlen_q, max_keys, tiles, splits, split_steps);
    const TalkPrefillArgs a{(const __bf16*)q, q_stride, (const __bf16*)keys, (const __bf16*)values, (int)key_pad, (int)vdim_pad, block_table,
                            bt_stride, (int)table_cols, (int)block_size, (int)num_blocks, seqs, cu_q, cu_k, (int)heads, (int)kv_heads, (int)dim,
                            (int)vdim, (int)num_seqs, 0, scale * kLog2e, (const __bf16*)talk, out_scale, (__bf16*)out, out_stride, workspace, tokens, splits,
                            split_steps, workspace + (heads * tokens + 3) / 4 * 4};
    hipStream_t st = (hipStream_t)stream;
    const bool bounded = max_score * kLog2e <= kBound;
    if (dim <= 64) return vdim <= 64 ? launch<2, 4>(a, max_seqlen_q, bounded, tiles, st) : launch<2, 8>(a, max_seqlen_q, bounded, tiles, st);
    return vdim <= 64 ? launch<4, 4>(a, max_seqlen_q, bounded, tiles, st) : launch<4, 8>(a, max_seqlen_q, bounded, tiles, st);
}
