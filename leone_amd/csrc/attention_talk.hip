// Attention whose heads' scores are mixed before the softmax, score_h <- sum_g talk[h, g] score_g, on the matrix cores,
// bfloat16 with float scores: both kernels hold the scores of all query heads of a piece of work in one wave's registers,
// in an order in which a float matrix instruction mixes them where they lie.
//
//   attention_talk_decode   one workgroup takes a query row, all its heads and one split of the keys; its four waves walk
//       tiles of 32 keys.  S [heads x keys] = Q K^T with v_mfma_f32_16x16x32_bf16, the rows of the other kv heads'
//       queries zero, so that every kv head's product adds into one tile of scores.  A lane (c, g) then holds key c and
//       heads 4 g .. 4 g + 3, one a register: register r is the operand "heads 4 g + r" of v_mfma_f32_16x16x4_f32, and four
//       of those are the mix.  The weights cross to the layout of O^T += V^T P^T through a wave's own piece of shared memory.
//   attention_talk_prefill  one workgroup takes 16 consecutive rows of a request, all heads, and walks the keys 64 or 128 at
//       a time, a wave 16 of them: S^T [keys x rows] of every head, so that a lane holds one row and four keys and every head
//       a register: v_mfma_f32_4x4x1_16b_f32 with its first operand broadcast (a column of talk) mixes them, four
//       heads an instruction (more than 16 heads: two workgroups make half the results each, the scores come sixteen heads
//       at a time and each sixteen add their part of the mix).  The weights go to shared memory, and for O^T += V^T P^T a
//       wave takes its share of the heads over all the stage's keys.
//
// The softmax is that of the other kernels: powers of two against a reference that is a whole number, raised only when a
// score outgrows it by 2^8; row sums over the rounded weights.  talk comes times scale * log2(e), in float.
#include "attention_merge.h"
#include "common.h"
#include "leone_hip.h"

#include <math.h>

namespace leone {

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8;
typedef __attribute__((__vector_size__(2 * sizeof(__bf16)))) __bf16 bf16x2;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;

constexpr int kTalkThreads = 256;
constexpr int kTalkWaves = 4;
constexpr float kTalkRaise = 8.0f;
constexpr float kLog2e = 1.4426950408889634f;

__device__ inline bf16x8 tk_load(const bf16_t* p) { return __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(p)); }
__device__ inline bf16x8 tk_zero() { return __builtin_bit_cast(bf16x8, uint4{0u, 0u, 0u, 0u}); }
// Two floats rounded to bfloat16, the first in the low half.
__device__ inline unsigned tk_pack(float a, float b) {
    const bf16x2 two = {static_cast<__bf16>(a), static_cast<__bf16>(b)};
    return __builtin_bit_cast(unsigned, two);
}
// Keeps the low or high half of every word where the key it belongs to is one that counts.
__device__ inline bf16x8 tk_keep(bf16x8 v, int first_key, int lo, int n) {
    uint4 raw = __builtin_bit_cast(uint4, v);
    unsigned* w = reinterpret_cast<unsigned*>(&raw);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int e0 = first_key + 2 * i, e1 = e0 + 1;
        unsigned mask = 0u;
        if (e0 >= lo && e0 < n) mask |= 0x0000ffffu;
        if (e1 >= lo && e1 < n) mask |= 0xffff0000u;
        w[i] &= mask;
    }
    return __builtin_bit_cast(bf16x8, raw);
}

// ---- single rows -------------------------------------------------------------------------------------------------
constexpr int kTalkRowStride = 40;         // elements from head to head of a wave's weights in shared memory (32 keys and room)

struct TalkArgs {
    const bf16_t* q;
    const bf16_t* k_pool;
    const bf16_t* v_pool;
    AnyVec talk;
    const int* positions;
    const int* block_table;
    int max_blocks;
    float* part_acc;
    float* part_ml;
    bf16_t* out;
    int q_heads, kv_heads, head_dim, v_dim, page_shift;
    float to_log2;
    int splits;
};

template <int kSize, int kHT>
__global__ void __launch_bounds__(kTalkThreads, 1)
attention_talk_decode_kernel(TalkArgs a, const int* __restrict__ row_entry, int window) {
    constexpr int kSteps = kSize / 32;                   // 32-element steps of a key
    constexpr int kVT = kSize / 16;                      // 16-element tiles of a value
    constexpr int kRing = 4;                             // pieces of keys or values on their way
    extern __shared__ float talk_lds[];
    const int heads = a.q_heads, kv_heads = a.kv_heads, group = heads / kv_heads;
    const int row = blockIdx.x, split = blockIdx.y;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave), lane = threadIdx.x % kWave;
    const int c = lane & 15, g = lane >> 4;
    const int page_tokens = 1 << a.page_shift, page_mask = page_tokens - 1;
    float* sm_acc = talk_lds;                                                            // [waves][heads][v_dim]
    float* sm_m = sm_acc + kTalkWaves * heads * a.v_dim;                                 // [waves][16 kHT]
    float* sm_l = sm_m + kTalkWaves * 16 * kHT;
    bf16_t* weights = reinterpret_cast<bf16_t*>(sm_l + kTalkWaves * 16 * kHT);           // [waves][kHT][16][kTalkRowStride]
    int* pages = reinterpret_cast<int*>(weights + kTalkWaves * kHT * 16 * kTalkRowStride);
    bf16_t* mine = weights + wave * kHT * 16 * kTalkRowStride;

    const int n = a.positions[row] + 1;
    const int lo = (window > 0 && n - window > 0) ? n - window : 0;
    const int t_begin = lo / 32, t_end = (n + 31) / 32;
    const int per_split = (t_end - t_begin + a.splits - 1) / a.splits;
    const int my_begin = t_begin + split * per_split;
    const int my_end = my_begin + per_split < t_end ? my_begin + per_split : t_end;
    const int* table = a.block_table + static_cast<long>(row_entry[row]) * a.max_blocks;
    const int first_page = (my_begin * 32) >> a.page_shift;
    if (my_begin < my_end) {
        const int last_key = (my_end * 32 < n ? my_end * 32 : n) - 1;
        const int count = (last_key >> a.page_shift) - first_page + 1;
        for (int i = threadIdx.x; i < count; i += kTalkThreads) pages[i] = table[first_page + i];
    }
    __syncthreads();

    // queries: row c of tile t is head 16 t + c, elements 32 s + 8 g ..; the mix's operands
    bf16x8 qreg[kHT][kSteps];
    int kv_of[kHT];                                       // the kv head of this lane's head (as a row and as a column)
    float mix[kHT][kHT][4];
#pragma unroll
    for (int t = 0; t < kHT; ++t) {
        const int h = 16 * t + c;
        kv_of[t] = h < heads ? h / group : -1;
        const bf16_t* from = a.q + (static_cast<long>(row) * heads + (h < heads ? h : 0)) * a.head_dim;
#pragma unroll
        for (int s = 0; s < kSteps; ++s) {
            const int at = 32 * s + 8 * g;
            qreg[t][s] = (h < heads && at < a.head_dim) ? tk_load(from + at) : tk_zero();
        }
#pragma unroll
        for (int u = 0; u < kHT; ++u)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int in = 16 * u + 4 * g + r;
                mix[t][u][r] = (h < heads && in < heads) ? load_any(a.talk, static_cast<long>(h) * heads + in) * a.to_log2 : 0.f;
            }
    }

    float m_run[kHT][4], l_run[kHT][4];
    floatx4 acc[kHT][kVT];
#pragma unroll
    for (int t = 0; t < kHT; ++t) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            m_run[t][r] = -INFINITY;
            l_run[t][r] = 0.f;
        }
#pragma unroll
        for (int dt = 0; dt < kVT; ++dt) acc[t][dt] = floatx4{0.f, 0.f, 0.f, 0.f};
    }
    bool unmapped = false;

    // A wave's work is a list of pieces: for every tile the keys of each kv head, then the values of each.  Every call of
    // `issue` gives the same number of loads (a piece that does not exist reads the pool's first page and is not used).
    bf16x8 ring[kRing][kVT];
    int ahead_tile = my_begin + wave, ahead_piece = 0;
    auto issue = [&](bf16x8* to) {
        const bool exists = ahead_tile < my_end;
        const int key0 = exists ? ahead_tile * 32 : 0;
        const bool keys = ahead_piece < kv_heads;
        const int kvh = !exists ? 0 : keys ? ahead_piece : ahead_piece - kv_heads;
        if (keys) {
#pragma unroll
            for (int half = 0; half < 2; ++half) {
                const int key = key0 + 16 * half;             // sixteen keys lie in one page
                int page = exists && key < n ? pages[(key >> a.page_shift) - first_page] : 0;
                if (page < 0) page = 0;
                const bf16_t* from = a.k_pool + (static_cast<long>(page) * kv_heads + kvh) * page_tokens * a.head_dim +
                                     static_cast<long>((key & page_mask) + c) * 8;
#pragma unroll
                for (int s = 0; s < kSteps; ++s) {
                    const int run = 32 * s + 8 * g < a.head_dim ? 4 * s + g : 0;
                    to[half * kSteps + s] = tk_load(from + static_cast<long>(run) * page_tokens * 8);
                }
            }
        } else {
            const int key = key0 + 8 * g;
            int page = exists && key < n ? pages[(key >> a.page_shift) - first_page] : 0;
            if (page < 0) page = 0;
            const bf16_t* from = a.v_pool + (static_cast<long>(page) * kv_heads + kvh) * page_tokens * a.v_dim +
                                 static_cast<long>((key & page_mask) >> 3) * a.v_dim * 8;
#pragma unroll
            for (int dt = 0; dt < kVT; ++dt) {
                const int d = 16 * dt + c < a.v_dim ? 16 * dt + c : 0;
                to[dt] = tk_load(from + static_cast<long>(d) * 8);
            }
        }
        if (++ahead_piece == 2 * kv_heads) {
            ahead_piece = 0;
            ahead_tile += kTalkWaves;
        }
    };

    floatx4 sc[kHT][2];
    bf16x8 pt[kHT];
    int tile = my_begin + wave, piece = 0;
    auto finish = [&](bf16x8* from) {
        const int key0 = tile * 32;
        const bool full = key0 >= lo && key0 + 32 <= n;
        if (piece < kv_heads) {
            if (piece == 0) {
#pragma unroll
                for (int t = 0; t < kHT; ++t) sc[t][0] = sc[t][1] = floatx4{0.f, 0.f, 0.f, 0.f};
            }
#pragma unroll
            for (int t = 0; t < kHT; ++t) {
                if ((piece + 1) * group <= 16 * t || piece * group >= 16 * (t + 1)) continue;       // no head of this kv head
#pragma unroll
                for (int s = 0; s < kSteps; ++s) {
                    const bf16x8 rows = kv_of[t] == piece ? qreg[t][s] : tk_zero();
                    sc[t][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(rows, from[s], sc[t][0], 0, 0, 0);
                    sc[t][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(rows, from[kSteps + s], sc[t][1], 0, 0, 0);
                }
            }
            if (piece == kv_heads - 1) {
                // lane (c, g): scores of key c (and 16 + c) for heads 16 t + 4 g + r.  Mixed, masked, weighed.
                floatx4 mixed[kHT][2];
#pragma unroll
                for (int t = 0; t < kHT; ++t)
#pragma unroll
                    for (int half = 0; half < 2; ++half) {
                        floatx4 sum = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                        for (int u = 0; u < kHT; ++u)
#pragma unroll
                            for (int r = 0; r < 4; ++r)
                                sum = __builtin_amdgcn_mfma_f32_16x16x4f32(mix[t][u][r], sc[u][half][r], sum, 0, 0, 0);
                        const int key = key0 + 16 * half + c;
                        if (!full && !(key >= lo && key < n)) sum = floatx4{-INFINITY, -INFINITY, -INFINITY, -INFINITY};
                        mixed[t][half] = sum;
                    }
                if (pages[(key0 >> a.page_shift) - first_page] < 0 ||
                    (key0 + 16 < n && pages[((key0 + 16) >> a.page_shift) - first_page] < 0))
                    unmapped = true;                          // the result is poisoned below
                bool raise = false;
#pragma unroll
                for (int t = 0; t < kHT; ++t)
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        raise = raise || fmaxf(mixed[t][0][r], mixed[t][1][r]) > m_run[t][r] + kTalkRaise;
                if (__any(raise)) {
#pragma unroll
                    for (int t = 0; t < kHT; ++t) {
                        float alpha[4];
#pragma unroll
                        for (int r = 0; r < 4; ++r) {
                            float top = fmaxf(mixed[t][0][r], mixed[t][1][r]);
#pragma unroll
                            for (int off = 1; off < 16; off <<= 1) top = fmaxf(top, __shfl_xor(top, off, kWave));
                            const float m_new = fmaxf(m_run[t][r], ceilf(top));
                            alpha[r] = m_new == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(m_run[t][r] - m_new);
                            m_run[t][r] = m_new;
                            l_run[t][r] *= alpha[r];
                        }
                        // the sums' columns are heads: column c's factor sits in the lanes of group c / 4, register c % 4
                        float factor = 0.f;
#pragma unroll
                        for (int r = 0; r < 4; ++r) {
                            const float got = __shfl(alpha[r], (c >> 2) * 16, kWave);
                            if ((c & 3) == r) factor = got;
                        }
#pragma unroll
                        for (int dt = 0; dt < kVT; ++dt)
#pragma unroll
                            for (int r = 0; r < 4; ++r) acc[t][dt][r] *= factor;
                    }
                }
#pragma unroll
                for (int t = 0; t < kHT; ++t)
#pragma unroll
                    for (int half = 0; half < 2; ++half)
#pragma unroll
                        for (int r = 0; r < 4; ++r) {
                            const float ref = m_run[t][r] == -INFINITY ? 0.f : m_run[t][r];
                            const __bf16 weight = static_cast<__bf16>(__builtin_amdgcn_exp2f(mixed[t][half][r] - ref));
                            l_run[t][r] += static_cast<float>(weight);
                            mine[(t * 16 + 4 * g + r) * kTalkRowStride + 16 * half + c].bits = __builtin_bit_cast(uint16_t, weight);
                        }
                __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
                __builtin_amdgcn_wave_barrier();
#pragma unroll
                for (int t = 0; t < kHT; ++t) pt[t] = tk_load(mine + (t * 16 + c) * kTalkRowStride + 8 * g);
                __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
                __builtin_amdgcn_wave_barrier();
            }
        } else {
            const int kvh = piece - kv_heads;
            if (!full) {                                      // slots outside the keys may hold anything, even NaN
#pragma unroll
                for (int dt = 0; dt < kVT; ++dt) from[dt] = tk_keep(from[dt], key0 + 8 * g, lo, n);
            }
#pragma unroll
            for (int t = 0; t < kHT; ++t) {
                if ((kvh + 1) * group <= 16 * t || kvh * group >= 16 * (t + 1)) continue;
                const bf16x8 columns = kv_of[t] == kvh ? pt[t] : tk_zero();
#pragma unroll
                for (int dt = 0; dt < kVT; ++dt) acc[t][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(from[dt], columns, acc[t][dt], 0, 0, 0);
            }
        }
        if (++piece == 2 * kv_heads) {
            piece = 0;
            tile += kTalkWaves;
        }
    };

    if (tile < my_end) {
#pragma unroll
        for (int i = 0; i < kRing; ++i) issue(ring[i]);
        while (true) {
            bool more = true;
#pragma unroll
            for (int i = 0; i < kRing; ++i) {
                if (more) {
                    finish(ring[i]);
                    issue(ring[i]);
                    more = tile < my_end;
                }
            }
            if (!more) break;
        }
    }

    // ---- merge the four waves
#pragma unroll
    for (int t = 0; t < kHT; ++t) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            float l = l_run[t][r];
#pragma unroll
            for (int off = 1; off < 16; off <<= 1) l += __shfl_xor(l, off, kWave);
            if (unmapped) l = __builtin_nanf("");
            if (c == 0) {
                sm_m[wave * 16 * kHT + 16 * t + 4 * g + r] = m_run[t][r];
                sm_l[wave * 16 * kHT + 16 * t + 4 * g + r] = l;
            }
        }
        const int h = 16 * t + c;
        if (h < heads) {
#pragma unroll
            for (int dt = 0; dt < kVT; ++dt)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int d = 16 * dt + 4 * g + r;
                    if (d < a.v_dim) sm_acc[(static_cast<long>(wave) * heads + h) * a.v_dim + d] = acc[t][dt][r];
                }
        }
    }
    __syncthreads();
    for (int i = threadIdx.x; i < heads * a.v_dim; i += kTalkThreads) {
        const int h = i / a.v_dim, d = i % a.v_dim;
        float top = -INFINITY;
#pragma unroll
        for (int w = 0; w < kTalkWaves; ++w) top = fmaxf(top, sm_m[w * 16 * kHT + h]);
        float num = 0.f, den = 0.f;
        if (top != -INFINITY) {
#pragma unroll
            for (int w = 0; w < kTalkWaves; ++w) {
                const float mw = sm_m[w * 16 * kHT + h];
                const float weight = mw == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(mw - top);
                num += sm_acc[(static_cast<long>(w) * heads + h) * a.v_dim + d] * weight;
                den += sm_l[w * 16 * kHT + h] * weight;
            }
        }
        const long rh = static_cast<long>(row) * heads + h;
        if (a.splits == 1) {
            a.out[rh * a.v_dim + d] = from_float<bf16_t>(num / den);
            continue;
        }
        const long slot = rh * a.splits + split;
        a.part_acc[slot * a.v_dim + d] = num;
        if (d == 0) {
            a.part_ml[slot * 2] = top;
            a.part_ml[slot * 2 + 1] = den;
        }
    }
}

static size_t talk_decode_shared(int heads, int v_dim, int tiles, int max_blocks) {
    return (static_cast<size_t>(kTalkWaves) * heads * v_dim + 2 * kTalkWaves * 16 * tiles) * sizeof(float) +
           static_cast<size_t>(kTalkWaves) * tiles * 16 * kTalkRowStride * sizeof(bf16_t) + static_cast<size_t>(max_blocks) * sizeof(int);
}

constexpr size_t kTalkMostShared = 160 * 1024;

// ---- tiles of rows -----------------------------------------------------------------------------------------------
constexpr int kTalkRows = 16;
// A workgroup takes all heads' scores and makes the results of the heads in `blocks` blocks of four: of all of them, or, with
// more than sixteen heads, of sixteen (another workgroup of the same rows makes the others).
// Waves of a workgroup: two a SIMD where there are heads enough for each to have its own and their scores fit beside them.
__host__ __device__ constexpr int talk_waves(int in_heads, int blocks) { return blocks == 1 || in_heads > 16 ? 4 : 8; }
// Turns in which the weights pass through shared memory: two where the queries of all heads take most of it.
__host__ __device__ constexpr int talk_turns(int size, int in_heads) { return in_heads > 16 && size > 64 ? 2 : 1; }

template <int kSize, int kIn, int kHB>
__host__ __device__ constexpr size_t talk_prefill_fixed() {
    // queries [heads][kSize / 8 runs][16 rows], weights [heads of a turn][2 runs a wave][16 rows] (16-byte runs),
    // maxima [waves][heads][16], references [heads][16], flags
    return static_cast<size_t>(kIn) * (kSize / 8) * 16 * 16 +
           static_cast<size_t>(4 * kHB / talk_turns(kSize, kIn)) * 2 * talk_waves(kIn, kHB) * 16 * 16 +
           static_cast<size_t>(talk_waves(kIn, kHB) + 1) * 4 * kHB * 16 * 4 + 16;
}

// kIn: heads whose scores are made (those beyond q_heads are zero).  kHB: blocks of four heads whose results are made, from
// head 4 kHB blockIdx.z on.  kLG: heads that share one load of keys.
template <int kSize, int kIn, int kHB, int kLG>
__global__ void __launch_bounds__(talk_waves(kIn, kHB) * kWave, talk_waves(kIn, kHB) / 4)
attention_talk_prefill_kernel(TalkArgs a, const int* __restrict__ tiles, int n_tiles) {
    constexpr int kH = 4 * kHB;
    constexpr int kSteps = kSize / 32, kVT = kSize / 16, kRuns = kSize / 8;
    constexpr int kLoads = kIn / kLG;                        // loads of keys a stage
    constexpr int kRing = kLoads < 2 ? kLoads : 2;
    constexpr int kWaves = talk_waves(kIn, kHB), kThreads = kWaves * kWave;
    constexpr int kStage = 16 * kWaves;                      // keys of a stage: sixteen a wave
    constexpr int kHW = kH / kWaves;                         // heads of a wave in the second product
    constexpr int kTurns = talk_turns(kSize, kIn), kHT = kHW / kTurns;   // heads of a wave in a turn
    constexpr int kPG = kLG < kHT ? kLG : kHT;               // of these, how many share one load of values
    constexpr int kHalves = kStage / 64;                     // the second product takes 64 keys at a time
    constexpr int kPRuns = kStage / 8;
    constexpr int kMixRegs = (kIn + 15) / 16;
    // More than sixteen heads: their scores come sixteen at a time, and the mixed ones are kept.  Otherwise the scores are
    // kept, and mixed anew where references are raised.
    constexpr bool kKeep = kIn > 16;
    constexpr int kScores = kKeep ? 16 : kIn;
    extern __shared__ uint4 talk_shared[];
    uint4* sq = talk_shared;                                 // [head][run][row]
    uint4* sp = sq + kIn * kRuns * 16;                       // [head of a turn][run of 8 keys][row]
    float* smax = reinterpret_cast<float*>(sp + kH / kTurns * kPRuns * 16);   // [wave][head][row]
    float* sref = smax + kWaves * kH * 16;                      // [head][row]
    int* flags = reinterpret_cast<int*>(sref + kH * 16);        // [2] raise, [2] unmapped
    int* pages = flags + 4;

    const int heads = a.q_heads, kv_heads = a.kv_heads, group = heads / kv_heads;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave), lane = threadIdx.x % kWave, tid = threadIdx.x;
    const int c = lane & 15, g = lane >> 4, out0 = kH * blockIdx.z;
    auto head_of = [&](int w) { return w / kHT * (kH / kTurns) + wave * kHT + w % kHT; };   // this wave's heads, from out0 on
    const int page_tokens = 1 << a.page_shift, page_mask = page_tokens - 1;
    const int* my_tile = tiles + 3 * static_cast<long>(n_tiles - 1 - static_cast<int>(blockIdx.x));   // the longest first
    const int entry = my_tile[0], row0 = my_tile[1], rows = my_tile[2];
    if (rows <= 0) return;
    const int p0 = a.positions[row0], p_last = p0 + rows - 1, n = p_last + 1;
    const int row_pos = c < rows ? p0 + c : -1;              // -1: sees no key
    const int split = blockIdx.y;
    const int stages = (n + kStage - 1) / kStage;
    const int share = (stages + a.splits - 1) / a.splits;
    const int st_begin = split * share, st_end = st_begin + share < stages ? st_begin + share : stages;
    if (st_begin >= st_end) {                                // more parts than stages: nothing of this one
        for (int i = tid; i < rows * kH; i += kThreads) {
            if (out0 + i % kH >= heads) continue;
            const long slot = ((static_cast<long>(row0) + i / kH) * heads + out0 + i % kH) * a.splits + split;
            a.part_ml[2 * slot] = -INFINITY;
            a.part_ml[2 * slot + 1] = 0.f;
        }
        return;
    }
    const int key_begin = st_begin * kStage, key_end = st_end * kStage < n ? st_end * kStage : n;
    const int first_page = key_begin >> a.page_shift;
    const int n_pages = ((key_end - 1) >> a.page_shift) - first_page + 1;
    const int* table = a.block_table + static_cast<long>(entry) * a.max_blocks;
    for (int i = tid; i < n_pages; i += kThreads) pages[i] = table[first_page + i];
    if (tid < 4) flags[tid] = 0;
    for (int i = tid; i < kH * 16; i += kThreads) sref[i] = -INFINITY;
    for (int i = tid; i < kIn * kRuns * 16; i += kThreads) {
        const int r = i % 16, run = (i / 16) % kRuns, h = i / (16 * kRuns);
        sq[i] = (h < heads && r < rows && 8 * run < a.head_dim)
                    ? *reinterpret_cast<const uint4*>(a.q + ((static_cast<long>(row0) + r) * heads + h) * a.head_dim + 8 * run)
                    : uint4{0u, 0u, 0u, 0u};
    }
    // the mix, four output heads and sixteen input heads a register: lane 4 b + i holds talk[out0 + 4 block + i][16 part + b]
    float mix[kHB][kMixRegs];
#pragma unroll
    for (int b = 0; b < kHB; ++b)
#pragma unroll
        for (int part = 0; part < kMixRegs; ++part) {
            const int to = out0 + 4 * b + (lane & 3), in = 16 * part + (lane >> 2);
            mix[b][part] = (to < heads && in < heads) ? load_any(a.talk, static_cast<long>(to) * heads + in) * a.to_log2 : 0.f;
        }
    __syncthreads();

    auto page_of = [&](int key) {                             // a page that is not there reads page 0 and poisons the result
        const int page = key < n ? pages[(key >> a.page_shift) - first_page] : 0;
        return page;
    };
    bf16x8 kx[kRing][kSteps];
    auto fetch_keys = [&](int st, int load, bf16x8* to) {
        const bool exists = st < st_end;
        const int key = exists ? st * kStage + 16 * wave : key_begin;
        const int page = page_of(key);
        int kvh = load * kLG / group;
        kvh = kvh < kv_heads ? kvh : kv_heads - 1;
        const bf16_t* from = a.k_pool + (static_cast<long>(page < 0 ? 0 : page) * kv_heads + kvh) * page_tokens * a.head_dim +
                             static_cast<long>((key & page_mask) + c) * 8;
#pragma unroll
        for (int s = 0; s < kSteps; ++s) {
            const int run = 32 * s + 8 * g < a.head_dim ? 4 * s + g : 0;
            to[s] = tk_load(from + static_cast<long>(run) * page_tokens * 8);
        }
    };
    bf16x8 vx[2][kVT];
    auto fetch_values = [&](int st, int half, int h) {
        int kvh = (out0 + h) / group;
        kvh = kvh < kv_heads ? kvh : kv_heads - 1;
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
            const int key = st * kStage + 64 * half + 32 * ks + 8 * g;
            const int page = page_of(key);
            const bf16_t* from = a.v_pool + (static_cast<long>(page < 0 ? 0 : page) * kv_heads + kvh) * page_tokens * a.v_dim +
                                 static_cast<long>((key & page_mask) >> 3) * a.v_dim * 8;
#pragma unroll
            for (int dt = 0; dt < kVT; ++dt) {
                const int d = 16 * dt + c < a.v_dim ? 16 * dt + c : 0;
                vx[ks][dt] = tk_load(from + static_cast<long>(d) * 8);
            }
        }
    };

    // where this lane's queries lie: an offset of a read reaches over sixteen heads and no further, so every sixteen have a
    // start of their own, which the compiler must not turn back into one for every read
    int q_at[kMixRegs];
#pragma unroll
    for (int part = 0; part < kMixRegs; ++part) {
        q_at[part] = 16 * (16 * part * kRuns + g) + c;
        if (part > 0) asm volatile("" : "+v"(q_at[part]));
    }
    float l_run[kHW];
    floatx4 acc[kHW][kVT];
#pragma unroll
    for (int w = 0; w < kHW; ++w) {
        l_run[w] = 0.f;
#pragma unroll
        for (int dt = 0; dt < kVT; ++dt) acc[w][dt] = floatx4{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int i = 0; i < kRing; ++i) fetch_keys(st_begin, i, kx[i]);

    for (int st = st_begin; st < st_end; ++st) {
        // ---- S^T of every head: lane (c, g) gets row c's scores of keys 4 g + r of this wave's sixteen
        floatx4 sc[kScores];
        floatx4 kept[kKeep ? kHB : 1][4];
        if constexpr (kKeep) {
#pragma unroll
            for (int b = 0; b < kHB; ++b)
#pragma unroll
                for (int r = 0; r < 4; ++r) kept[b][r] = floatx4{0.f, 0.f, 0.f, 0.f};
        }
#define LEONE_TALK_ONE(PART, I)                                                                                                   \
    if constexpr (16 * (PART) + (I) < kIn) {                                                                                      \
        _Pragma("unroll") for (int r = 0; r < 4; ++r)                                                                             \
            d[r] = __builtin_amdgcn_mfma_f32_4x4x1f32(mix[b][PART], sc[(16 * (PART) + (I)) % kScores][r], d[r], 4, I, 0);         \
    }
#define LEONE_TALK_FOUR(PART, I) LEONE_TALK_ONE(PART, I) LEONE_TALK_ONE(PART, I + 1) LEONE_TALK_ONE(PART, I + 2) LEONE_TALK_ONE(PART, I + 3)
#define LEONE_TALK_SIXTEEN(PART) LEONE_TALK_FOUR(PART, 0) LEONE_TALK_FOUR(PART, 4) LEONE_TALK_FOUR(PART, 8) LEONE_TALK_FOUR(PART, 12)
#pragma unroll
        for (int load = 0; load < kLoads; ++load) {
            bf16x8* keys = kx[load % kRing];
#pragma unroll
            for (int i = 0; i < kLG; ++i) {
                const int h = load * kLG + i;
                floatx4 sum = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int s = 0; s < kSteps; ++s)
                    sum = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                        keys[s], __builtin_bit_cast(bf16x8, sq[q_at[h / 16] + (h % 16 * kRuns + 4 * s) * 16]), sum, 0, 0, 0);
                sc[h % kScores] = sum;
                if constexpr (kKeep) __builtin_amdgcn_sched_barrier(0);      // or queries far ahead take the registers
            }
            // the ring's next piece: a later load of this stage, or one of the next stage's first
            fetch_keys(load + kRing < kLoads ? st : st + 1, (load + kRing) % kLoads, keys);
            if constexpr (kKeep) {                            // sixteen heads' scores are there: their part of the mix
                __builtin_amdgcn_sched_barrier(0);
                if ((load + 1) * kLG % 16 == 0) {
#pragma unroll
                    for (int b = 0; b < kHB; ++b) {
                        floatx4* d = kept[b];
                        if (load * kLG / 16 == 0) {
                            LEONE_TALK_SIXTEEN(0)
                        } else {
                            if constexpr (kMixRegs > 1) { LEONE_TALK_SIXTEEN(1) }
                        }
                    }
                    __builtin_amdgcn_sched_barrier(0);
                }
            }
        }

        // ---- mixed scores and weights of all heads
        const int key0 = st * kStage + 16 * wave + 4 * g;
        const bool full = (st + 1) * kStage <= p0 + 1;
        uint2 packed[kH];
        int* flag = flags + (st & 1);
        bool maxima = st == st_begin;                         // the first scores always raise the references
        bool met = false;                                     // the workgroup has met behind the stage before
        while (true) {                                        // every wave takes the same turns
            bool raise = false;
#pragma unroll
            for (int b = 0; b < kHB; ++b) {
                floatx4 d[4];                                 // d[r][i]: head 4 b + i, key 4 g + r
#pragma unroll
                for (int r = 0; r < 4; ++r) d[r] = kKeep ? kept[kKeep ? b : 0][r] : floatx4{0.f, 0.f, 0.f, 0.f};
                if constexpr (!kKeep) { LEONE_TALK_SIXTEEN(0) }
                if (!full) {
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        if (key0 + r > row_pos) d[r] = floatx4{-INFINITY, -INFINITY, -INFINITY, -INFINITY};
                }
                if (maxima) {
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        float top = fmaxf(fmaxf(d[0][i], d[1][i]), fmaxf(d[2][i], d[3][i]));
                        top = fmaxf(top, __shfl_xor(top, 16, kWave));
                        top = fmaxf(top, __shfl_xor(top, 32, kWave));
                        if (g == 0) smax[(wave * kH + 4 * b + i) * 16 + c] = top;
                    }
                } else {
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        const int h = 4 * b + i;
                        float ref = sref[h * 16 + c];
                        raise = raise || fmaxf(fmaxf(d[0][i], d[1][i]), fmaxf(d[2][i], d[3][i])) > ref + kTalkRaise;
                        ref = ref == -INFINITY ? 0.f : ref;
                        packed[h].x = tk_pack(__builtin_amdgcn_exp2f(d[0][i] - ref), __builtin_amdgcn_exp2f(d[1][i] - ref));
                        packed[h].y = tk_pack(__builtin_amdgcn_exp2f(d[2][i] - ref), __builtin_amdgcn_exp2f(d[3][i] - ref));
                    }
                }
                __builtin_amdgcn_sched_barrier(0);            // block by block: all of them at once do not fit the registers
            }
            if (!maxima) {
                if (met) break;
                if (__any(raise) && lane == 0) *flag = 1;
                __syncthreads();                              // the weights of the stage before have been read
                met = true;
                if (*flag == 0) break;
                maxima = true;
                continue;
            }
            __syncthreads();
            met = true;
            maxima = false;
            // a wave raises the references of its own heads and carries its sums over
#pragma unroll
            for (int w = 0; w < kHW; ++w) {
                const int h = head_of(w);
                float top = smax[h * 16 + c];
#pragma unroll
                for (int v = 1; v < kWaves; ++v) top = fmaxf(top, smax[(v * kH + h) * 16 + c]);
                const float before = sref[h * 16 + c];
                const float m_new = fmaxf(before, ceilf(top));
                const float alpha = m_new == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(before - m_new);
                if (g == 0) sref[h * 16 + c] = m_new;
                l_run[w] *= alpha;
#pragma unroll
                for (int dt = 0; dt < kVT; ++dt)
#pragma unroll
                    for (int r = 0; r < 4; ++r) acc[w][dt][r] *= alpha;
            }
            __syncthreads();
        }
        if (page_of(st * kStage + 16 * wave) < 0) flags[2] = 1;
        if (tid == 0) flags[(st & 1) ^ 1] = 0;                // the next stage's flag: it is set behind the barrier below
#undef LEONE_TALK_SIXTEEN
#undef LEONE_TALK_FOUR
#undef LEONE_TALK_ONE
        // ---- O^T += V^T P^T: this wave's heads over all of the stage's keys
#pragma unroll
        for (int turn = 0; turn < kTurns; ++turn) {
            if constexpr (kTurns > 1) __builtin_amdgcn_sched_barrier(0);     // or both turns' values are asked for at once
            fetch_values(st, 0, head_of(turn * kHT));
            if (turn > 0) __syncthreads();                    // the weights of the turn before have been read
#pragma unroll
            for (int h = 0; h < kH / kTurns; ++h)
                reinterpret_cast<uint2*>(sp)[((h * kPRuns + 2 * wave + (g >> 1)) * 16 + c) * 2 + (g & 1)] = packed[turn * (kH / kTurns) + h];
            __syncthreads();
#pragma unroll
            for (int half = 0; half < kHalves; ++half) {
                const int begin = st * kStage + 64 * half;
                if (begin >= n) continue;                     // the same for the workgroup
                const bool whole = begin + 64 <= n;
#pragma unroll
                for (int w0 = 0; w0 < kHT; w0 += kPG) {
                    if (half + w0 > 0) fetch_values(st, half, head_of(turn * kHT + w0));
                    if (!whole) {                             // slots behind the keys may hold anything, even NaN
#pragma unroll
                        for (int ks = 0; ks < 2; ++ks)
#pragma unroll
                            for (int dt = 0; dt < kVT; ++dt) vx[ks][dt] = tk_keep(vx[ks][dt], begin + 32 * ks + 8 * g, 0, n);
                    }
#pragma unroll
                    for (int i = 0; i < kPG; ++i) {
                        const int w = turn * kHT + w0 + i, h = wave * kHT + w0 + i;
#pragma unroll
                        for (int ks = 0; ks < 2; ++ks) {
                            const uint4 raw = sp[(h * kPRuns + 8 * half + 4 * ks + g) * 16 + c];
                            const bf16x8 pt = __builtin_bit_cast(bf16x8, raw);
                            const unsigned pairs[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
                            for (int j = 0; j < 4; ++j)
                                l_run[w] = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2, pairs[j]),
                                                                           __builtin_bit_cast(bf16x2, 0x3f803f80u), l_run[w], false);
#pragma unroll
                            for (int dt = 0; dt < kVT; ++dt) acc[w][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vx[ks][dt], pt, acc[w][dt], 0, 0, 0);
                        }
                    }
                }
            }
        }
    }
    const bool poisoned = flags[2] != 0;                      // every write came before the last barrier
#pragma unroll
    for (int w = 0; w < kHW; ++w) {
        const int h = head_of(w);
        float l = l_run[w];
        l += __shfl_xor(l, 16, kWave);
        l += __shfl_xor(l, 32, kWave);
        if (poisoned) l = __builtin_nanf("");
        if (out0 + h >= heads || c >= rows) continue;
        const long rh = (static_cast<long>(row0) + c) * heads + out0 + h;
        if (a.splits > 1) {
            const float ref = sref[h * 16 + c];
            const long slot = rh * a.splits + split;
            if (g == 0) {
                a.part_ml[2 * slot] = ref;
                a.part_ml[2 * slot + 1] = l;
            }
#pragma unroll
            for (int dt = 0; dt < kVT; ++dt)
                if (16 * dt + 4 * g < a.v_dim) *reinterpret_cast<floatx4*>(a.part_acc + slot * a.v_dim + 16 * dt + 4 * g) = acc[w][dt];
            continue;
        }
        const float inv = 1.0f / l;
#pragma unroll
        for (int dt = 0; dt < kVT; ++dt) {
            const int d = 16 * dt + 4 * g;
            if (d >= a.v_dim) continue;
            uint2 two;
            two.x = tk_pack(acc[w][dt][0] * inv, acc[w][dt][1] * inv);
            two.y = tk_pack(acc[w][dt][2] * inv, acc[w][dt][3] * inv);
            *reinterpret_cast<uint2*>(a.out + rh * a.v_dim + d) = two;
        }
    }
}

static int raise_shared(const void* kernel, size_t bytes, size_t* allowed, const char* what) {
    if (bytes <= *allowed) return 0;
    const hipError_t e = hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(bytes));
    if (e != hipSuccess) {
        set_error("%s: %zu bytes of shared memory were refused: %s", what, bytes, hipGetErrorString(e));
        return 1;
    }
    *allowed = bytes;
    return 0;
}

static int check_talk(const char* what, const TalkArgs& a, int page_tokens, int talk_dtype, int most_heads) {
    LEONE_REQUIRE(a.q && a.out && a.k_pool && a.v_pool && a.talk.ptr && a.positions && a.block_table, "%s: null pointer", what);
    LEONE_REQUIRE(talk_dtype == kF32 || talk_dtype == kBF16, "%s: unknown type of the mix", what);
    LEONE_REQUIRE(a.q_heads > 0 && a.q_heads <= most_heads && a.kv_heads > 0 && a.q_heads % a.kv_heads == 0,
                  "%s: %d query heads (at most %d) over %d kv heads", what, a.q_heads, most_heads, a.kv_heads);
    LEONE_REQUIRE(a.head_dim > 0 && a.head_dim % 8 == 0 && a.head_dim <= 128 && a.v_dim > 0 && a.v_dim % 4 == 0 && a.v_dim <= 128,
                  "%s: heads of %d (a multiple of 8 up to 128) and values of %d elements (a multiple of 4 up to 128)", what, a.head_dim, a.v_dim);
    LEONE_REQUIRE(page_tokens >= 16 && (page_tokens & (page_tokens - 1)) == 0 && a.max_blocks > 0,
                  "%s: page_tokens %d must be a power of two, at least 16", what, page_tokens);
    LEONE_REQUIRE(a.splits >= 1 && (a.splits == 1 || (a.part_acc && a.part_ml)), "%s: %d splits need the workspace", what, a.splits);
    return 0;
}

static int shift_of(int page_tokens) {
    int shift = 0;
    while ((1 << shift) < page_tokens) ++shift;
    return shift;
}

}  // namespace leone

using namespace leone;

extern "C" int leone_attention_talk_tile_rows() { return kTalkRows; }

// bfloat16, up to 32 query heads, heads of a multiple of 8 and values of a multiple of 4 elements up to 128, pages of a
// power of two of at least 16 tokens.  Workspace for splits > 1: part_acc rows * q_heads * splits * v_dim floats, part_ml
// rows * q_heads * splits * 2.
extern "C" int leone_attention_talk_decode(const void* q, void* out, const void* k_pool, const void* v_pool, const void* talk,
                                           int talk_dtype, const int* positions, const int* row_entry, const int* block_table,
                                           int max_blocks, float* part_acc, float* part_ml, int rows, int q_heads, int kv_heads,
                                           int head_dim, int v_dim, int page_tokens, float scale, int window, int splits,
                                           hipStream_t stream) {
    const TalkArgs a{static_cast<const bf16_t*>(q), static_cast<const bf16_t*>(k_pool), static_cast<const bf16_t*>(v_pool),
                     AnyVec{talk, talk_dtype}, positions, block_table, max_blocks, part_acc, part_ml, static_cast<bf16_t*>(out),
                     q_heads, kv_heads, head_dim, v_dim, shift_of(page_tokens), scale * kLog2e, splits};
    if (check_talk("attention_talk_decode", a, page_tokens, talk_dtype, 32)) return 1;
    LEONE_REQUIRE(row_entry && rows > 0 && window >= 0 && splits <= attention_reduce_max_splits(),
                  "attention_talk_decode: rows %d, window %d, splits %d", rows, window, splits);
    const int tiles = q_heads <= 16 ? 1 : 2;
    const size_t shared = talk_decode_shared(q_heads, v_dim, tiles, max_blocks);
    LEONE_REQUIRE(shared <= kTalkMostShared, "attention_talk_decode: %zu bytes of shared memory are too many", shared);
    const int size = head_dim > v_dim ? head_dim : v_dim;
#define LEONE_TALK_DECODE(SIZE, HT)                                                                                               \
    do {                                                                                                                          \
        static size_t allowed = 48 * 1024;                                                                                        \
        if (raise_shared(reinterpret_cast<const void*>(&attention_talk_decode_kernel<SIZE, HT>), shared, &allowed,                \
                         "attention_talk_decode"))                                                                                \
            return 1;                                                                                                             \
        attention_talk_decode_kernel<SIZE, HT><<<dim3(rows, splits), kTalkThreads, shared, stream>>>(a, row_entry, window);       \
    } while (0)
    if (size <= 32) {
        if (tiles == 1) LEONE_TALK_DECODE(32, 1); else LEONE_TALK_DECODE(32, 2);
    } else if (size <= 64) {
        if (tiles == 1) LEONE_TALK_DECODE(64, 1); else LEONE_TALK_DECODE(64, 2);
    } else {
        if (tiles == 1) LEONE_TALK_DECODE(128, 1); else LEONE_TALK_DECODE(128, 2);
    }
#undef LEONE_TALK_DECODE
    LEONE_LAUNCH_CHECK("attention_talk_decode");
    if (splits > 1) {
        launch_attention_reduce(part_acc, part_ml, static_cast<bf16_t*>(out), rows, q_heads, v_dim, splits, stream);
        LEONE_LAUNCH_CHECK("attention_talk_decode merge");
    }
    return 0;
}

// tiles int32 [n_tiles, 3]: (entry, first row, rows) with at most leone_attention_talk_tile_rows() consecutive rows of one
// request; otherwise as above.  Workspace for splits > 1: part_acc covered rows * q_heads * splits *
// v_dim floats, part_ml covered rows * q_heads * splits * 2, `covered rows` one more than the last row a tile names.
extern "C" int leone_attention_talk_prefill(const void* q, void* out, const void* k_pool, const void* v_pool, const void* talk,
                                            int talk_dtype, const int* positions, const int* tiles, int n_tiles,
                                            const int* block_table, int max_blocks, float* part_acc, float* part_ml, int q_heads,
                                            int kv_heads, int head_dim, int v_dim, int page_tokens, float scale, int splits,
                                            hipStream_t stream) {
    const TalkArgs a{static_cast<const bf16_t*>(q), static_cast<const bf16_t*>(k_pool), static_cast<const bf16_t*>(v_pool),
                     AnyVec{talk, talk_dtype}, positions, block_table, max_blocks, part_acc, part_ml, static_cast<bf16_t*>(out),
                     q_heads, kv_heads, head_dim, v_dim, shift_of(page_tokens), scale * kLog2e, splits};
    if (check_talk("attention_talk_prefill", a, page_tokens, talk_dtype, 32)) return 1;
    LEONE_REQUIRE(tiles && n_tiles > 0 && splits <= attention_tile_merge_max_splits(), "attention_talk_prefill: %d tiles, splits %d", n_tiles, splits);
    const int size = head_dim > v_dim ? head_dim : v_dim;
    const bool grouped = (q_heads / kv_heads) % 4 == 0;       // four neighbouring heads read the same keys
#define LEONE_TALK_PREFILL(SIZE, IN, HB, LG)                                                                                      \
    do {                                                                                                                          \
        static size_t allowed = 48 * 1024;                                                                                        \
        const size_t shared = talk_prefill_fixed<SIZE, IN, HB>() + static_cast<size_t>(max_blocks) * sizeof(int);                 \
        LEONE_REQUIRE(shared <= kTalkMostShared, "attention_talk_prefill: %zu bytes of shared memory are too many", shared);      \
        if (raise_shared(reinterpret_cast<const void*>(&attention_talk_prefill_kernel<SIZE, IN, HB, LG>), shared, &allowed,       \
                         "attention_talk_prefill"))                                                                               \
            return 1;                                                                                                             \
        attention_talk_prefill_kernel<SIZE, IN, HB, LG><<<dim3(n_tiles, splits, ceil_div(q_heads, 4 * HB)),                       \
                                                          talk_waves(IN, HB) * kWave, shared, stream>>>(a, tiles, n_tiles);       \
    } while (0)
#define LEONE_TALK_SIZES(IN, HB)                                                            \
    if (size <= 64) {                                                                       \
        if (grouped) LEONE_TALK_PREFILL(64, IN, HB, 4); else LEONE_TALK_PREFILL(64, IN, HB, 1);    \
    } else {                                                                                \
        if (grouped) LEONE_TALK_PREFILL(128, IN, HB, 4); else LEONE_TALK_PREFILL(128, IN, HB, 1);  \
    }
    if (q_heads <= 4) {
        LEONE_TALK_SIZES(4, 1)
    } else if (q_heads <= 8) {
        LEONE_TALK_SIZES(8, 2)
    } else if (q_heads <= 16) {
        LEONE_TALK_SIZES(16, 4)
    } else {
        LEONE_TALK_SIZES(32, 4)
    }
#undef LEONE_TALK_SIZES
#undef LEONE_TALK_PREFILL
    LEONE_LAUNCH_CHECK("attention_talk_prefill");
    if (splits > 1) {
        launch_attention_tile_merge(part_acc, part_ml, static_cast<bf16_t*>(out), tiles, n_tiles, q_heads, v_dim, splits, stream);
        LEONE_LAUNCH_CHECK("attention_talk_prefill merge");
    }
    return 0;
}
