// What stands ahead of a matrix memory whose projections read the token before beside the token itself:
//
//   token_mix       out[m, r] = h[r] + (h[r'] - h[r]) * mu[m] for `mixes` vectors mu, r' the row of the token before: the
//                   row above within a portion, the request's stored row ahead of one, zeros at a sequence's start.  The
//                   last row of every entry becomes the request's stored row (float).
//   low_rank_decay  w[r, c] = exp(-exp(sum_i w2[c, i] * tanh(low[r, i]) + w0[c])), all of it float.
//
// The memory itself is time_mix_scan in gated_scan.hip.
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

// A workgroup takes kRows rows and 64 * kCols channels; its four waves share out the rank, a lane holds kCols channels (64
// apart) of every row, the rows' tanh values are made once.  The waves' sums meet in shared memory in their order.
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
        const dim3 grid(ceil_div(rows, 16), ceil_div(channels, 2 * kWave));
        LEONE_REQUIRE(grid.y <= 65535, "low_rank_decay: too many channels");
        low_rank_decay_kernel<16, 2><<<grid, kMixThreads, 0, stream>>>(low, low_stride, matrix, base, out, rows, channels, rank, runs);
    }
    LEONE_LAUNCH_CHECK("low_rank_decay");
    return 0;
}
