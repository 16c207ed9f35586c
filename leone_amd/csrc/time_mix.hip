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
#pragma unroll
    for (int i = 0; i < kRun; ++i) {
        own[i] = to_float(h[at + i]);
        before[i] = 0.f;
    }
    if (row > span[0]) {
#pragma unroll
        for (int i = 0; i < kRun; ++i) before[i] = to_float(h[at - hidden + i]);
    } else if (span[2] >= 0) {
        const float* from = state + static_cast<long>(span[2]) * hidden + c;
#pragma unroll
        for (int i = 0; i < kRun; ++i) before[i] = from[i];
    }
    for (int m = 0; m < mixes; ++m) {
        T* to = out + static_cast<long>(m) * rows * hidden + at;
#pragma unroll
        for (int i = 0; i < kRun; ++i) to[i] = from_float<T>(fmaf(before[i] - own[i], load_any(mu, static_cast<long>(m) * hidden + c + i), own[i]));
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

// A workgroup takes kDecayRows rows and 256 channels, a thread one channel; the rows' tanh values are made once.
constexpr int kDecayRows = 8;

__global__ void __launch_bounds__(kMixThreads)
low_rank_decay_kernel(const float* __restrict__ low, long low_stride, AnyVec w2, AnyVec w0, float* __restrict__ out, int rows,
                      int channels, int rank) {
    extern __shared__ float bent[];                            // [rank][kDecayRows]
    const int row0 = blockIdx.x * kDecayRows;
    const int here = rows - row0 < kDecayRows ? rows - row0 : kDecayRows;
    for (int i = threadIdx.x; i < kDecayRows * rank; i += kMixThreads) {
        const int r = i / rank, k = i % rank;
        bent[k * kDecayRows + r] = r < here ? tanhf(low[static_cast<long>(row0 + r) * low_stride + k]) : 0.f;
    }
    __syncthreads();
    const int c = blockIdx.y * kMixThreads + threadIdx.x;
    if (c >= channels) return;
    float sum[kDecayRows];
    const float base = load_any(w0, c);
#pragma unroll
    for (int r = 0; r < kDecayRows; ++r) sum[r] = 0.f;
    const long at = static_cast<long>(c) * rank;
    int k = 0;
    if (rank % 8 == 0) {
        for (; k < rank; k += 8) {
            float w[8];
            load_any8(w2, at + k, w);
#pragma unroll
            for (int i = 0; i < 8; ++i)
#pragma unroll
                for (int r = 0; r < kDecayRows; ++r) sum[r] = fmaf(w[i], bent[(k + i) * kDecayRows + r], sum[r]);
        }
    }
    for (; k < rank; ++k) {
        const float w = load_any(w2, at + k);
#pragma unroll
        for (int r = 0; r < kDecayRows; ++r) sum[r] = fmaf(w, bent[k * kDecayRows + r], sum[r]);
    }
#pragma unroll
    for (int r = 0; r < kDecayRows; ++r)
        if (r < here) out[static_cast<long>(row0 + r) * channels + c] = expf(-expf(sum[r] + base));
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
    const int run = hidden % 4 == 0 && rows >= 64 ? 4 : 1;
    const dim3 grid(rows, ceil_div(hidden, kMixThreads * run));
    LEONE_REQUIRE(grid.y <= 65535, "token_mix: rows of %d are too wide", hidden);
#define LEONE_TOKEN_MIX(T, RUN)                                                                                                  \
    token_mix_kernel<T, RUN><<<grid, kMixThreads, 0, stream>>>(static_cast<const T*>(h), AnyVec{mu, mu_dtype}, mixes, state,       \
                                                               state_out, spans, row_entry, static_cast<T*>(out), rows, hidden,   \
                                                               single_rows)
    if (dtype == kF32) {
        if (run == 4) LEONE_TOKEN_MIX(float, 4);
        else LEONE_TOKEN_MIX(float, 1);
    } else {
        if (run == 4) LEONE_TOKEN_MIX(bf16_t, 4);
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
    const size_t shared = static_cast<size_t>(kDecayRows) * rank * sizeof(float);
    LEONE_REQUIRE(shared <= 60 * 1024, "low_rank_decay: a rank of %d does not fit shared memory", rank);
    LEONE_REQUIRE(rank % 8 != 0 || reinterpret_cast<uintptr_t>(w2) % 32 == 0, "low_rank_decay: the matrix must be aligned to 32 bytes");
    const dim3 grid(ceil_div(rows, kDecayRows), ceil_div(channels, kMixThreads));
    LEONE_REQUIRE(grid.y <= 65535, "low_rank_decay: too many channels");
    low_rank_decay_kernel<<<grid, kMixThreads, shared, stream>>>(low, low_stride, AnyVec{w2, w2_dtype}, AnyVec{w0, w0_dtype}, out, rows,
                                                                 channels, rank);
    LEONE_LAUNCH_CHECK("low_rank_decay");
    return 0;
}
