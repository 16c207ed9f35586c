// A matrix memory whose projections read the token before beside the token itself and whose decays come from the token:
//
//   token_mix       out[m, r] = h[r] + (h[r'] - h[r]) * mu[m] for `mixes` vectors mu, r' the row of the token before: the
//                   row above within a portion, the request's stored row ahead of one, zeros at a sequence's start.  The
//                   last row of every entry becomes the request's stored row (float).
//   low_rank_decay  w[r, c] = exp(-exp(sum_i w2[c, i] * tanh(low[r, i]) + w0[c])), all of it float.
//
//   time_mix_scan   per head o_t = (S + diag(bonus) k_t v_t^T)^T r_t, then S <- diag(w_t) S + k_t v_t^T, row by row.  A wave
//                   owns a run of columns of one head of one segment (a request's rows in the step, or a chunk of them): a
//                   column's key channels are spread over 1 to 16 neighbouring lanes, 16 a lane, four columns a lane; r, w and
//                   k of 8 rows at a time lie in shared memory, the next 8 rows' are on their way meanwhile; the lanes of
//                   a column add their parts of a read-out by moves within a row of lanes.
//   time_mix_read   long portions: chunks are walked side by side from zeros, their end states chained (gated_chain), and what a
//                   chunk's rows read of the state the chunk starts from is one product for all rows.
//
// Everything in the memory is float.
#include "common.h"
#include "leone_hip.h"

#include <math.h>

namespace leone {

constexpr int kMixThreads = 256;
constexpr int kMixMost = 8;

template <typename T, int kRun>
__device__ inline void mix_load(const T* p, float* to) {
    if constexpr (kRun == 8) {
        load_any8(AnyVec{p, sizeof(T) == 4 ? kF32 : kBF16}, 0, to);
    } else {
        to[0] = to_float(*p);
    }
}
template <typename T, int kRun>
__device__ inline void mix_store(T* p, const float* v) {
    if constexpr (kRun == 8 && sizeof(T) == 2) {
        uint4 raw;
        unsigned* w = reinterpret_cast<unsigned*>(&raw);
#pragma unroll
        for (int i = 0; i < 4; ++i) w[i] = bf16_bits_from_float(v[2 * i]) | (static_cast<unsigned>(bf16_bits_from_float(v[2 * i + 1])) << 16);
        *reinterpret_cast<uint4*>(p) = raw;
    } else if constexpr (kRun == 8) {
        reinterpret_cast<float4*>(p)[0] = float4{v[0], v[1], v[2], v[3]};
        reinterpret_cast<float4*>(p)[1] = float4{v[4], v[5], v[6], v[7]};
    } else {
        *p = from_float<T>(v[0]);
    }
}

// spans [entries][4]: first row, end, slot read (negative: a sequence's start), slot written.
template <typename T, int kRun>
__global__ void __launch_bounds__(kMixThreads)
token_mix_kernel(const T* __restrict__ h, AnyVec mu, int mixes, const float* __restrict__ state, float* __restrict__ state_out,
                 const int* __restrict__ spans, const int* __restrict__ row_entry, T* __restrict__ out, int rows, int hidden,
                 int single_rows) {
    const int row = blockIdx.x;
    const int c = (blockIdx.y * kMixThreads + threadIdx.x) * kRun;
    if (c >= hidden) return;
    const int* span = spans + 4 * row_entry[row];
    const long at = static_cast<long>(row) * hidden + c;
    float own[kRun], before[kRun];
    mix_load<T, kRun>(h + at, own);
#pragma unroll
    for (int i = 0; i < kRun; ++i) before[i] = 0.f;
    if (row > span[0]) mix_load<T, kRun>(h + at - hidden, before);
    else if (span[2] >= 0) mix_load<float, kRun>(state + static_cast<long>(span[2]) * hidden + c, before);
#pragma unroll
    for (int m = 0; m < kMixMost; ++m) {
        if (m >= mixes) break;
        float share[kRun], mixed[kRun];
        if constexpr (kRun == 8) load_any8(mu, static_cast<long>(m) * hidden + c, share);
        else share[0] = load_any(mu, static_cast<long>(m) * hidden + c);
#pragma unroll
        for (int i = 0; i < kRun; ++i) mixed[i] = fmaf(before[i] - own[i], share[i], own[i]);
        mix_store<T, kRun>(out + static_cast<long>(m) * rows * hidden + at, mixed);
    }
    // a step of single rows: nobody else reads this entry's stored row
    if (single_rows && state_out != nullptr) {
        float* to = state_out + static_cast<long>(span[3]) * hidden + c;
#pragma unroll
        for (int i = 0; i < kRun; ++i) to[i] = own[i];
    }
}

template <typename T>
__global__ void __launch_bounds__(kMixThreads)
token_mix_keep_kernel(const T* __restrict__ h, float* __restrict__ state_out, const int* __restrict__ spans, int hidden) {
    const int* span = spans + 4 * blockIdx.x;
    const int c = blockIdx.y * kMixThreads + threadIdx.x;
    if (c >= hidden || span[1] <= span[0]) return;
    state_out[static_cast<long>(span[3]) * hidden + c] = to_float(h[static_cast<long>(span[1] - 1) * hidden + c]);
}

// Few rows: a workgroup takes kRows rows and 64 * kCols channels; its four waves share out the rank, a lane holds kCols
// channels (64 apart) of every row, the rows' tanh values are made once.  The waves' sums meet in shared memory in their order.
constexpr int kDecayRank = 64;              // ranks worked off at a time

template <int kRows, int kCols>
__global__ void __launch_bounds__(kMixThreads)
low_rank_decay_kernel(const float* __restrict__ low, long low_stride, AnyVec w2, AnyVec w0, float* __restrict__ out, int rows,
                      int channels, int rank, int runs) {
    __shared__ __align__(16) float bent[kDecayRank * kRows];           // [rank][row]
    __shared__ float part[kMixThreads / kWave][kRows][kCols][kWave];
    const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
    const int row0 = blockIdx.x * kRows;
    const int here = rows - row0 < kRows ? rows - row0 : kRows;
    int ch[kCols];
#pragma unroll
    for (int j = 0; j < kCols; ++j) ch[j] = blockIdx.y * kWave * kCols + j * kWave + lane;
    float sum[kRows][kCols];
#pragma unroll
    for (int r = 0; r < kRows; ++r)
#pragma unroll
        for (int j = 0; j < kCols; ++j) sum[r][j] = 0.f;
    constexpr int kShare = kDecayRank / (kMixThreads / kWave);          // ranks a wave takes of those at hand
    for (int k0 = 0; k0 < rank; k0 += kDecayRank) {
        // the matrix is asked for before the tanh values are made: neither waits for the other
        float w[kCols][kShare];
        const int first = k0 + wave * kShare;
#pragma unroll
        for (int j = 0; j < kCols; ++j) {
            const long at = static_cast<long>(ch[j] < channels ? ch[j] : channels - 1) * rank + first;
            if (runs && first + kShare <= rank) {
#pragma unroll
                for (int i = 0; i < kShare; i += 8) load_any8(w2, at + i, w[j] + i);
            } else {
#pragma unroll
                for (int i = 0; i < kShare; ++i) w[j][i] = first + i < rank ? load_any(w2, at + i) : 0.f;
            }
        }
        __syncthreads();
        for (int i = threadIdx.x; i < kDecayRank * kRows; i += kMixThreads) {
            const int r = i / kDecayRank, k = i % kDecayRank;
            bent[k * kRows + r] = (r < here && k0 + k < rank) ? tanhf(low[static_cast<long>(row0 + r) * low_stride + k0 + k]) : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int i = 0; i < kShare; ++i)
#pragma unroll
            for (int r = 0; r < kRows; ++r) {
                const float b = bent[(wave * kShare + i) * kRows + r];
#pragma unroll
                for (int j = 0; j < kCols; ++j) sum[r][j] = fmaf(w[j][i], b, sum[r][j]);
            }
    }
#pragma unroll
    for (int r = 0; r < kRows; ++r)
#pragma unroll
        for (int j = 0; j < kCols; ++j) part[wave][r][j][lane] = sum[r][j];
    __syncthreads();
    for (int i = threadIdx.x; i < kRows * kCols * kWave; i += kMixThreads) {
        const int l = i % kWave, j = (i / kWave) % kCols, r = i / (kWave * kCols);
        const int c = blockIdx.y * kWave * kCols + j * kWave + l;
        if (r >= here || c >= channels) continue;
        float total = load_any(w0, c);
#pragma unroll
        for (int v = 0; v < kMixThreads / kWave; ++v) total += part[v][r][j][l];
        out[static_cast<long>(row0 + r) * channels + c] = expf(-expf(total));
    }
}

// The same for many rows: a workgroup takes 64 rows and 128 channels, a lane two channels with their whole rows of the
// matrix in registers (up to kDecayRank elements at a time), a wave 16 rows.
constexpr int kDecayTile = 64;

__global__ void __launch_bounds__(kMixThreads)
low_rank_decay_rows_kernel(const float* __restrict__ low, long low_stride, AnyVec w2, AnyVec w0, float* __restrict__ out, int rows,
                           int channels, int rank, int runs) {
    constexpr int kRank = 32;                                          // of the rank at a time
    constexpr int kRows = kDecayTile / (kMixThreads / kWave);
    __shared__ __align__(16) float bent[kDecayTile][kRank];
    const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
    const int row0 = blockIdx.x * kDecayTile;
    const int ch[2] = {static_cast<int>(blockIdx.y) * 2 * kWave + lane, static_cast<int>(blockIdx.y) * 2 * kWave + kWave + lane};
    float sum[kRows][2];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
        const float base = ch[j] < channels ? load_any(w0, ch[j]) : 0.f;
#pragma unroll
        for (int r = 0; r < kRows; ++r) sum[r][j] = base;
    }
    for (int k0 = 0; k0 < rank; k0 += kRank) {
        float w[2][kRank];
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const long at = static_cast<long>(ch[j] < channels ? ch[j] : channels - 1) * rank + k0;
            if (runs && k0 + kRank <= rank) {
#pragma unroll
                for (int i = 0; i < kRank; i += 8) load_any8(w2, at + i, w[j] + i);
            } else {
#pragma unroll
                for (int i = 0; i < kRank; ++i) w[j][i] = k0 + i < rank ? load_any(w2, at + i) : 0.f;
            }
        }
        __syncthreads();
#pragma unroll
        for (int u = 0; u < kDecayTile * kRank / kMixThreads; ++u) {
            const int i = u * kMixThreads + threadIdx.x, r = i / kRank, k = i % kRank;
            bent[r][k] = (row0 + r < rows && k0 + k < rank) ? tanhf(low[static_cast<long>(row0 + r) * low_stride + k0 + k]) : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int r = 0; r < kRows; ++r)
#pragma unroll
            for (int i = 0; i < kRank; i += 4) {
                const float4 b = *reinterpret_cast<const float4*>(&bent[wave * kRows + r][i]);
#pragma unroll
                for (int j = 0; j < 2; ++j)
                    sum[r][j] = fmaf(w[j][i + 3], b.w, fmaf(w[j][i + 2], b.z, fmaf(w[j][i + 1], b.y, fmaf(w[j][i], b.x, sum[r][j]))));
            }
    }
#pragma unroll
    for (int r = 0; r < kRows; ++r) {
        const int row = row0 + wave * kRows + r;
        if (row >= rows) break;
#pragma unroll
        for (int j = 0; j < 2; ++j)
            if (ch[j] < channels) out[static_cast<long>(row) * channels + ch[j]] = expf(-expf(sum[r][j]));
    }
}

// ---- the memory --------------------------------------------------------------------------------------------------
struct MixSegment {
    int first, end, in, out;        // rows [first, end); state read (negative: zeros) and written (negative: nowhere)
};

constexpr int kScanRows = 16;       // key channels a lane holds
constexpr int kScanCols = 4;        // columns a lane holds: what it reads from shared memory serves all four
constexpr int kScanMaxDim = 256;

struct TimeMixArgs {
    const float* r;                 // [rows, stride], head h at h * dim; k likewise, v at h * vdim
    const float* k;
    const float* v;
    long stride;
    const float* decay;             // [rows, heads * dim]
    AnyVec bonus;                   // [heads * dim]
    const MixSegment* segments;
    const float* state_in;          // [index, heads, dim * vdim]
    long in_stride;
    float* state_out;
    long out_stride;
    float* product;                 // [segments, heads, dim]: the product of the decays over a segment's rows, or null
    float* out;                     // [rows, heads, vdim]
    int heads, dim, vdim;
};

// Sum over kGroups neighbouring lanes; every one of them gets it.
template <int kGroups>
__device__ inline float lanes_sum(float v) {
    if constexpr (kGroups >= 2) v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xB1, 0xf, 0xf, true));    // 1 0 3 2
    if constexpr (kGroups >= 4) v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x4E, 0xf, 0xf, true));    // 2 3 0 1
    if constexpr (kGroups >= 8) v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x141, 0xf, 0xf, true));   // mirrored in eight
    if constexpr (kGroups >= 16) v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x140, 0xf, 0xf, true));  // mirrored in sixteen
    return v;
}

// kTokens rows are staged at a time (1: a step of single rows).  kRuns: vdim is a multiple of 4.
template <int kGroups, int kTokens, bool kTrack, bool kRuns>
__global__ void __launch_bounds__(256, 2) time_mix_scan_kernel(TimeMixArgs p) {
    constexpr int kDim = kGroups * kScanRows;                 // channels with those that fill up the last lane
    constexpr int kHold = kTokens == 1 ? (kDim + kWave - 1) / kWave : kTokens;    // staged elements a thread holds at most
    constexpr int kColLanes = kWave / kGroups;
    __shared__ __align__(16) float staged[3][kTokens][kDim];  // r, w, k
    const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, threads = blockDim.x;
    const MixSegment seg = p.segments[blockIdx.x];
    const int head = blockIdx.y;
    const int part = lane % kGroups, ch0 = part * kScanRows;
    const int col0 = ((blockIdx.z * (threads / kWave) + wave) * kColLanes + lane / kGroups) * kScanCols;
    const bool mine = col0 < p.vdim;
    const int n = seg.end - seg.first;
    if (n <= 0) return;

    auto columns = [&](const float* from, float* to) {        // four columns; those that do not exist repeat one that does
        if constexpr (kRuns) {
            const float4 v = *reinterpret_cast<const float4*>(from + (mine ? col0 : 0));
            to[0] = v.x, to[1] = v.y, to[2] = v.z, to[3] = v.w;
        } else {
#pragma unroll
            for (int c = 0; c < kScanCols; ++c) to[c] = from[col0 + c < p.vdim ? col0 + c : 0];
        }
    };
    float hold[3][kHold];
    auto ask = [&](int t0) {                                  // rows from t0 on into registers; rows that do not exist repeat the last
#pragma unroll
        for (int u = 0; u < kHold; ++u) {
            if (u * threads >= kTokens * kDim) break;
            const int e = u * threads + tid, t = t0 + e / kDim, i = e % kDim;
            const long row = seg.first + (t < n ? t : n - 1);
            const int ch = head * p.dim + (i < p.dim ? i : 0);
            hold[0][u] = p.r[row * p.stride + ch];
            hold[1][u] = p.decay[row * p.heads * p.dim + ch];
            hold[2][u] = p.k[row * p.stride + ch];
        }
    };
    ask(0);
    float S[kScanRows][kScanCols], u[kScanRows], carried = 1.f;    // carried: thread i follows channel i
#pragma unroll
    for (int i = 0; i < kScanRows; ++i) u[i] = load_any(p.bonus, head * p.dim + (ch0 + i < p.dim ? ch0 + i : 0));
    if (seg.in >= 0) {                                        // the same for the workgroup
        const float* from = p.state_in + seg.in * p.in_stride + static_cast<long>(head) * p.dim * p.vdim;
#pragma unroll
        for (int i = 0; i < kScanRows; ++i) columns(from + static_cast<long>(ch0 + i < p.dim ? ch0 + i : 0) * p.vdim, S[i]);
    } else {
#pragma unroll
        for (int i = 0; i < kScanRows; ++i)
#pragma unroll
            for (int c = 0; c < kScanCols; ++c) S[i][c] = 0.f;
    }
    float v_next[kScanCols];
    columns(p.v + static_cast<long>(seg.first) * p.stride + head * p.vdim, v_next);

    for (int t0 = 0; t0 < n; t0 += kTokens) {
        const int here = n - t0 < kTokens ? n - t0 : kTokens;
        __syncthreads();                                      // everyone is done with the rows before
#pragma unroll
        for (int w = 0; w < kHold; ++w) {
            const int e = w * threads + tid;
            if (e < kTokens * kDim) {
                const bool there = e % kDim < p.dim;          // channels that fill up the last lane carry and read nothing
                (&staged[0][0][0])[e] = there ? hold[0][w] : 0.f;
                (&staged[1][0][0])[e] = there ? hold[1][w] : 0.f;
                (&staged[2][0][0])[e] = there ? hold[2][w] : 0.f;
            }
        }
        __syncthreads();
        if (t0 + kTokens < n) ask(t0 + kTokens);
        for (int t = 0; t < here; ++t) {
            const long row = seg.first + t0 + t;
            float v[kScanCols], acc[kScanCols], now = 0.f;
#pragma unroll
            for (int c = 0; c < kScanCols; ++c) {
                v[c] = v_next[c];
                acc[c] = 0.f;
            }
            if constexpr (kTrack) carried *= staged[1][t][tid < kDim ? tid : 0];
            const long row_next = t0 + t + 1 < n ? row + 1 : row;
            columns(p.v + row_next * p.stride + head * p.vdim, v_next);
#pragma unroll
            for (int i0 = 0; i0 < kScanRows; i0 += 4) {
                const float4 qr = *reinterpret_cast<const float4*>(&staged[0][t][ch0 + i0]);
                const float4 wr = *reinterpret_cast<const float4*>(&staged[1][t][ch0 + i0]);
                const float4 kr = *reinterpret_cast<const float4*>(&staged[2][t][ch0 + i0]);
                const float q[4] = {qr.x, qr.y, qr.z, qr.w}, w[4] = {wr.x, wr.y, wr.z, wr.w}, k[4] = {kr.x, kr.y, kr.z, kr.w};
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const int i = i0 + j;
                    now = fmaf(u[i] * k[j], q[j], now);
#pragma unroll
                    for (int c = 0; c < kScanCols; ++c) {
                        acc[c] = fmaf(S[i][c], q[j], acc[c]);                 // the state before this row
                        S[i][c] = fmaf(w[j], S[i][c], k[j] * v[c]);
                    }
                }
            }
#pragma unroll
            for (int c = 0; c < kScanCols; ++c) acc[c] = lanes_sum<kGroups>(fmaf(now, v[c], acc[c]));
            if (part == 0 && mine) {
                float* to = p.out + (row * p.heads + head) * p.vdim + col0;
                if constexpr (kRuns) {
                    *reinterpret_cast<float4*>(to) = float4{acc[0], acc[1], acc[2], acc[3]};
                } else {
#pragma unroll
                    for (int c = 0; c < kScanCols; ++c)
                        if (col0 + c < p.vdim) to[c] = acc[c];
                }
            }
        }
    }
    if constexpr (kTrack) {
        if (p.product && blockIdx.z == 0 && tid < p.dim)
            p.product[(static_cast<long>(blockIdx.x) * p.heads + head) * p.dim + tid] = carried;
    }
    if (!p.state_out || seg.out < 0 || !mine) return;
    float* to = p.state_out + seg.out * p.out_stride + static_cast<long>(head) * p.dim * p.vdim;
#pragma unroll
    for (int i = 0; i < kScanRows; ++i) {
        if (ch0 + i >= p.dim) continue;
        float* row = to + static_cast<long>(ch0 + i) * p.vdim + col0;
        if constexpr (kRuns) {
            *reinterpret_cast<float4*>(row) = float4{S[i][0], S[i][1], S[i][2], S[i][3]};
        } else {
#pragma unroll
            for (int c = 0; c < kScanCols; ++c)
                if (col0 + c < p.vdim) row[c] = S[i][c];
        }
    }
}

template <int kGroups>
static void launch_time_mix_scan(const TimeMixArgs& a, int n_segments, bool single, hipStream_t stream) {
    constexpr int kPerWave = kWave / kGroups * kScanCols;
    int waves = ceil_div(a.vdim, kPerWave) < 4 ? ceil_div(a.vdim, kPerWave) : 4;
    const int least = kGroups * kScanRows / kWave;            // a thread then stages at most as many elements as rows are staged
    waves = waves < least ? least : waves;
    const dim3 grid(n_segments, a.heads, ceil_div(a.vdim, waves * kPerWave));
    const bool runs = a.vdim % 4 == 0 && a.stride % 4 == 0 && reinterpret_cast<uintptr_t>(a.v) % 16 == 0 &&
                      reinterpret_cast<uintptr_t>(a.out) % 16 == 0 && reinterpret_cast<uintptr_t>(a.state_in) % 16 == 0 &&
                      reinterpret_cast<uintptr_t>(a.state_out) % 16 == 0 && a.in_stride % 4 == 0 && a.out_stride % 4 == 0;
#define LEONE_TIME_MIX(TOKENS, TRACK)                                                                              \
    do {                                                                                                           \
        if (runs) time_mix_scan_kernel<kGroups, TOKENS, TRACK, true><<<grid, waves * kWave, 0, stream>>>(a);       \
        else time_mix_scan_kernel<kGroups, TOKENS, TRACK, false><<<grid, waves * kWave, 0, stream>>>(a);           \
    } while (0)
    if (a.product) LEONE_TIME_MIX(8, true);
    else if (single) LEONE_TIME_MIX(1, false);
    else LEONE_TIME_MIX(8, false);
#undef LEONE_TIME_MIX
}

// What the rows of a chunk read of the state S the chunk starts from, for the time-mixing form: nothing is written into S on
// the way, so row t reads S scaled by the product of the rows' decays before it, o_t += S^T (r_t * prod_(s < t) w_s), and
// all rows are one product.  A workgroup takes a segment (up to kReadRows rows) and a head; the scaled r of all rows lie
// channel by channel in shared memory, S comes by kReadDepth channels at a time, a thread holds 4 rows x 4 columns.
constexpr int kReadRows = 64;
constexpr int kReadCols = 64;
constexpr int kReadDepth = 32;

__global__ void __launch_bounds__(256)
time_mix_read_kernel(const float* __restrict__ r, long stride, const float* __restrict__ decay, const MixSegment* __restrict__ segments,
                     const float* __restrict__ state, long state_stride, float* __restrict__ out, int heads, int dim, int vdim) {
    extern __shared__ __align__(16) float read_lds[];
    float* scaled = read_lds;                                 // [dim][kReadRows]
    float* s_state = scaled + dim * kReadRows;                // [kReadDepth][kReadCols]
    const MixSegment seg = segments[blockIdx.x];
    const int head = blockIdx.y, tid = threadIdx.x;
    const int n = seg.end - seg.first;
    if (seg.in < 0) return;
    for (int i = tid; i < dim; i += 256) {
        const float* rp = r + static_cast<long>(seg.first) * stride + head * dim + i;
        const float* wp = decay + (static_cast<long>(seg.first) * heads + head) * dim + i;
        float before = 1.f;
#pragma unroll 8
        for (int t = 0; t < kReadRows; ++t) {
            const int at = t < n ? t : n - 1;                 // rows beyond the segment are not stored
            scaled[i * kReadRows + t] = rp[at * stride] * before;
            before *= wp[static_cast<long>(at) * heads * dim];
        }
    }
    const int row0 = (tid / 16) * 4, col0 = (tid % 16) * 4;
    const float* from = state + seg.in * state_stride + static_cast<long>(head) * dim * vdim;
    for (int base = 0; base < vdim; base += kReadCols) {
        float sum[4][4];
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int j = 0; j < 4; ++j) sum[i][j] = 0.f;
        for (int d0 = 0; d0 < dim; d0 += kReadDepth) {
            __syncthreads();
            for (int i = tid; i < kReadDepth * kReadCols; i += 256) {
                const int d = d0 + i / kReadCols, c = base + i % kReadCols;
                s_state[i] = (d < dim && c < vdim) ? from[static_cast<long>(d) * vdim + c] : 0.f;
            }
            __syncthreads();
            const int depth = dim - d0 < kReadDepth ? dim - d0 : kReadDepth;
            for (int d = 0; d < depth; ++d) {
                const float4 a = *reinterpret_cast<const float4*>(scaled + (d0 + d) * kReadRows + row0);
                const float4 b = *reinterpret_cast<const float4*>(s_state + d * kReadCols + col0);
                const float av[4] = {a.x, a.y, a.z, a.w}, bv[4] = {b.x, b.y, b.z, b.w};
#pragma unroll
                for (int i = 0; i < 4; ++i)
#pragma unroll
                    for (int j = 0; j < 4; ++j) sum[i][j] = fmaf(av[i], bv[j], sum[i][j]);
            }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int t = row0 + i, c = base + col0 + j;
                if (t < n && c < vdim) out[((static_cast<long>(seg.first) + t) * heads + head) * vdim + c] += sum[i][j];
            }
    }
}

}  // namespace leone

using namespace leone;

extern "C" int leone_token_mix(const void* h, int dtype, const void* mu, int mu_dtype, int mixes, const float* state,
                               float* state_out, const int* spans, int entries, const int* row_entry, void* out, int rows,
                               int hidden, int single_rows, hipStream_t stream) {
    LEONE_REQUIRE((dtype == kF32 || dtype == kBF16) && (mu_dtype == kF32 || mu_dtype == kBF16), "token_mix: unknown element type");
    LEONE_REQUIRE(h && mu && state && spans && row_entry && out, "token_mix: null pointer");
    LEONE_REQUIRE(rows > 0 && hidden > 0 && entries > 0 && mixes > 0 && mixes <= kMixMost, "token_mix: %d rows of %d, %d entries, %d mixes",
                  rows, hidden, entries, mixes);
    LEONE_REQUIRE(!single_rows || rows == entries, "token_mix: %d rows of %d entries are no single rows", rows, entries);
    const bool aligned = reinterpret_cast<uintptr_t>(h) % 32 == 0 && reinterpret_cast<uintptr_t>(mu) % 32 == 0 &&
                         reinterpret_cast<uintptr_t>(state) % 32 == 0 && reinterpret_cast<uintptr_t>(out) % 32 == 0;
    const int run = hidden % 8 == 0 && aligned && rows >= 64 ? 8 : 1;
    const dim3 grid(rows, ceil_div(hidden, kMixThreads * run));
    LEONE_REQUIRE(grid.y <= 65535, "token_mix: rows of %d are too wide", hidden);
#define LEONE_TOKEN_MIX(T, RUN)                                                                                                  \
    token_mix_kernel<T, RUN><<<grid, kMixThreads, 0, stream>>>(static_cast<const T*>(h), AnyVec{mu, mu_dtype}, mixes, state,       \
                                                               state_out, spans, row_entry, static_cast<T*>(out), rows, hidden,   \
                                                               single_rows)
    if (dtype == kF32) {
        if (run == 8) LEONE_TOKEN_MIX(float, 8);
        else LEONE_TOKEN_MIX(float, 1);
    } else {
        if (run == 8) LEONE_TOKEN_MIX(bf16_t, 8);
        else LEONE_TOKEN_MIX(bf16_t, 1);
    }
#undef LEONE_TOKEN_MIX
    LEONE_LAUNCH_CHECK("token_mix");
    if (state_out && !single_rows) {
        const dim3 keep(entries, ceil_div(hidden, kMixThreads));
        if (dtype == kF32)
            token_mix_keep_kernel<float><<<keep, kMixThreads, 0, stream>>>(static_cast<const float*>(h), state_out, spans, hidden);
        else
            token_mix_keep_kernel<bf16_t><<<keep, kMixThreads, 0, stream>>>(static_cast<const bf16_t*>(h), state_out, spans, hidden);
        LEONE_LAUNCH_CHECK("token_mix_keep");
    }
    return 0;
}

extern "C" int leone_low_rank_decay(const float* low, long low_stride, const void* w2, int w2_dtype, const void* w0, int w0_dtype,
                                    float* out, int rows, int channels, int rank, hipStream_t stream) {
    LEONE_REQUIRE(low && w2 && w0 && out, "low_rank_decay: null pointer");
    LEONE_REQUIRE((w2_dtype == kF32 || w2_dtype == kBF16) && (w0_dtype == kF32 || w0_dtype == kBF16), "low_rank_decay: unknown element type");
    LEONE_REQUIRE(rows > 0 && channels > 0 && rank > 0 && low_stride >= rank, "low_rank_decay: %d rows, %d channels, rank %d", rows, channels, rank);
    const int runs = rank % 8 == 0 && reinterpret_cast<uintptr_t>(w2) % 32 == 0;
    const AnyVec matrix{w2, w2_dtype}, base{w0, w0_dtype};
    if (rows <= 64) {
        const dim3 grid(ceil_div(rows, 8), ceil_div(channels, kWave));
        LEONE_REQUIRE(grid.y <= 65535, "low_rank_decay: too many channels");
        low_rank_decay_kernel<8, 1><<<grid, kMixThreads, 0, stream>>>(low, low_stride, matrix, base, out, rows, channels, rank, runs);
    } else {
        const dim3 grid(ceil_div(rows, kDecayTile), ceil_div(channels, 2 * kWave));
        LEONE_REQUIRE(grid.y <= 65535, "low_rank_decay: too many channels");
        low_rank_decay_rows_kernel<<<grid, kMixThreads, 0, stream>>>(low, low_stride, matrix, base, out, rows, channels, rank, runs);
    }
    LEONE_LAUNCH_CHECK("low_rank_decay");
    return 0;
}

// r, k, v float [rows, stride] (heads * dim, heads * dim and heads * vdim columns), decay float [rows, heads * dim], bonus
// [heads * dim] of bonus_dtype; segments int32 [n, 4]: first row, end, index of the state read (negative: zeros), of the state
// written (negative: nowhere); states float [index, heads, dim * vdim] of the given strides (either may be null);
// decay_product (may be null) float [segments, heads, dim]; single_rows: every segment has at most one row.
extern "C" int leone_time_mix_scan(const float* r, const float* k, const float* v, long stride, const float* decay,
                                   const void* bonus, int bonus_dtype, const int* segments, int n_segments, int single_rows,
                                   const float* state_in, long in_stride, float* state_out, long out_stride,
                                   float* decay_product, float* out, int heads, int dim, int vdim, hipStream_t stream) {
    LEONE_REQUIRE(r && k && v && decay && bonus && segments && out, "time_mix_scan: null pointer");
    LEONE_REQUIRE(bonus_dtype == kF32 || bonus_dtype == kBF16, "time_mix_scan: unknown element type");
    LEONE_REQUIRE(n_segments > 0 && heads > 0 && heads <= 65535 && dim > 0 && dim <= kScanMaxDim && vdim > 0,
                  "time_mix_scan: %d segments, %d heads of %d (at most %d) x %d", n_segments, heads, dim, kScanMaxDim, vdim);
    const long per_slot = static_cast<long>(heads) * dim * vdim;
    LEONE_REQUIRE((!state_in || in_stride >= per_slot) && (!state_out || out_stride >= per_slot),
                  "time_mix_scan: states of %ld floats do not fit", per_slot);
    LEONE_REQUIRE(stride >= static_cast<long>(heads) * (dim > vdim ? dim : vdim), "time_mix_scan: rows of %ld do not hold the heads", stride);
    const TimeMixArgs a{r, k, v, stride, decay, AnyVec{bonus, bonus_dtype}, reinterpret_cast<const MixSegment*>(segments), state_in,
                        in_stride, state_out, out_stride, decay_product, out, heads, dim, vdim};
    const bool single = single_rows != 0;
    if (dim <= 16) launch_time_mix_scan<1>(a, n_segments, single, stream);
    else if (dim <= 32) launch_time_mix_scan<2>(a, n_segments, single, stream);
    else if (dim <= 64) launch_time_mix_scan<4>(a, n_segments, single, stream);
    else if (dim <= 128) launch_time_mix_scan<8>(a, n_segments, single, stream);
    else launch_time_mix_scan<16>(a, n_segments, single, stream);
    LEONE_LAUNCH_CHECK("time_mix_scan");
    return 0;
}

extern "C" int leone_time_mix_read_rows() { return kReadRows; }

// Adds to out what every segment's rows (at most leone_time_mix_read_rows() each) read of the state named by its third word.
extern "C" int leone_time_mix_read(const float* r, long stride, const float* decay, const int* segments, int n_segments,
                                   const float* state, long state_stride, float* out, int heads, int dim, int vdim, hipStream_t stream) {
    LEONE_REQUIRE(r && decay && segments && state && out, "time_mix_read: null pointer");
    LEONE_REQUIRE(n_segments > 0 && heads > 0 && heads <= 65535 && dim > 0 && dim <= kScanMaxDim && vdim > 0 &&
                      stride >= static_cast<long>(heads) * dim && state_stride >= static_cast<long>(heads) * dim * vdim,
                  "time_mix_read: %d segments, %d heads of %d x %d", n_segments, heads, dim, vdim);
    const size_t shared = (static_cast<size_t>(dim) * kReadRows + kReadDepth * kReadCols) * sizeof(float);
    static size_t allowed = 48 * 1024;
    if (shared > allowed) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&time_mix_read_kernel), hipFuncAttributeMaxDynamicSharedMemorySize,
                                                 static_cast<int>(shared));
        LEONE_REQUIRE(e == hipSuccess, "time_mix_read: %zu bytes of shared memory were refused: %s", shared, hipGetErrorString(e));
        allowed = shared;
    }
    time_mix_read_kernel<<<dim3(n_segments, heads), 256, shared, stream>>>(r, stride, decay, reinterpret_cast<const MixSegment*>(segments),
                                                                           state, state_stride, out, heads, dim, vdim);
    LEONE_LAUNCH_CHECK("time_mix_read");
    return 0;
}
