// What several sublayers that read the same stream add to it, and the norms that read the stream next, in one kernel:
//
//   branch_norm   x += sum_t factor_t * scale_t * rows_t   (rows_t float [n, hidden], or planes [p, n, hidden] whose sum, in
//                 order, is meant; scale_t a vector [hidden] or absent), then, for up to two norms,
//                 y = x * gain / sqrt(mean over the column's group of x^2 + eps), the columns in `groups` equal groups of
//                 neighbours.  With `picked` only those rows come out and x is left as it was.
//
//   stream_join   the same sum, then the operand [x | first] of a product that reads the stream beside another float tensor
//                 [n, hidden], in that product's type; x becomes a vector, the same for every row, to which the product is added.
//
// One workgroup a row; the row lies in shared memory between the passes, every wave sums squares of a group or of an equal
// share of one, and a group's shares are added in order, so a launch repeats bit for bit.  All sums are float.
#include "common.h"
#include "leone_hip.h"

#include <math.h>

namespace leone {

constexpr int kBranchTerms = 4;
constexpr int kBranchNorms = 2;
constexpr int kBranchMaxThreads = 1024;

struct BranchTerm {
    const float* rows;
    AnyVec scale;
    float factor;
    int planes;
    long plane;
};

struct BranchNormArgs {
    float* x;
    BranchTerm term[kBranchTerms];
    int terms;
    AnyVec gain[kBranchNorms];
    void* y[kBranchNorms];
    int norms;
    float eps;
    int groups;
    const int* picked;
    int hidden;
};

template <int kRun>
__device__ inline void load_run_f(const float* p, float* to) {
    if constexpr (kRun == 4) {
        const float4 v = *reinterpret_cast<const float4*>(p);
        to[0] = v.x, to[1] = v.y, to[2] = v.z, to[3] = v.w;
    } else {
        to[0] = *p;
    }
}

template <int kRun>
__device__ inline void load_run_any(const AnyVec& v, int at, float* to) {
    if constexpr (kRun == 4) {
        if (v.dtype == kF32) {
            load_run_f<4>(static_cast<const float*>(v.ptr) + at, to);
        } else {
            const uint2 raw = *reinterpret_cast<const uint2*>(static_cast<const bf16_t*>(v.ptr) + at);
            to[0] = __uint_as_float(raw.x << 16), to[1] = __uint_as_float(raw.x & 0xffff0000u);
            to[2] = __uint_as_float(raw.y << 16), to[3] = __uint_as_float(raw.y & 0xffff0000u);
        }
    } else {
        to[0] = load_any(v, at);
    }
}

// Columns c .. c + kRun - 1 of row `in_row` of the stream with all results added.
template <int kRun>
__device__ inline void summed_run(const float* xr, const BranchTerm* term, int terms, long in_row, int hidden, int c, float v[kRun]) {
    load_run_f<kRun>(xr + c, v);
#pragma unroll
    for (int t = 0; t < kBranchTerms; ++t) {
        if (t >= terms) break;
        const float* from = term[t].rows + in_row * hidden + c;
        float d[kRun], s[kRun];
        load_run_f<kRun>(from, d);
        for (int p = 1; p < term[t].planes; ++p) {
            float more[kRun];
            load_run_f<kRun>(from + p * term[t].plane, more);
#pragma unroll
            for (int i = 0; i < kRun; ++i) d[i] += more[i];
        }
        if (term[t].scale.ptr) {
            load_run_any<kRun>(term[t].scale, c, s);
#pragma unroll
            for (int i = 0; i < kRun; ++i) v[i] = fmaf(term[t].factor * s[i], d[i], v[i]);
        } else {
#pragma unroll
            for (int i = 0; i < kRun; ++i) v[i] = fmaf(term[t].factor, d[i], v[i]);
        }
    }
}

template <typename TY, int kRun>
__device__ inline void store_run(TY* to, const float v[kRun]) {
    if constexpr (kRun == 4 && sizeof(TY) == 2) {
        uint2 packed;
        packed.x = bf16_bits_from_float(v[0]) | (static_cast<uint32_t>(bf16_bits_from_float(v[1])) << 16);
        packed.y = bf16_bits_from_float(v[2]) | (static_cast<uint32_t>(bf16_bits_from_float(v[3])) << 16);
        *reinterpret_cast<uint2*>(to) = packed;
    } else if constexpr (kRun == 4) {
        *reinterpret_cast<float4*>(to) = float4{v[0], v[1], v[2], v[3]};
    } else {
        *to = from_float<TY>(v[0]);
    }
}

template <typename TY, int kRun>
__global__ void __launch_bounds__(kBranchMaxThreads) branch_norm_kernel(BranchNormArgs a) {
    extern __shared__ __align__(16) float branch_lds[];
    float* srow = branch_lds;                                  // [hidden]
    float* share_sum = srow + (a.hidden + 3) / 4 * 4;           // [groups * shares]
    const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, waves = blockDim.x / kWave;
    const long in_row = a.picked ? a.picked[blockIdx.x] : blockIdx.x;
    float* xr = a.x + in_row * a.hidden;
    const int step = blockDim.x * kRun;
#pragma unroll 2
    for (int c = tid * kRun; c < a.hidden; c += step) {
        float v[kRun];
        summed_run<kRun>(xr, a.term, a.terms, in_row, a.hidden, c, v);
#pragma unroll
        for (int i = 0; i < kRun; ++i) srow[c + i] = v[i];
        if (a.terms > 0 && !a.picked) store_run<float, kRun>(xr + c, v);
    }
    if (a.norms == 0) return;
    __syncthreads();
    // a group's columns in `shares` equal runs, one run a wave
    const int size = a.hidden / a.groups;
    const int shares = waves / a.groups > 1 ? waves / a.groups : 1;
    for (int item = wave; item < a.groups * shares; item += waves) {
        const int g = item / shares, s = item % shares;
        const int begin = static_cast<int>(static_cast<long>(size) * s / shares), end = static_cast<int>(static_cast<long>(size) * (s + 1) / shares);
        float ss = 0.f;
        for (int i = begin + lane; i < end; i += kWave) {
            const float v = srow[g * size + i];
            ss = fmaf(v, v, ss);
        }
        ss = wave_sum(ss);
        if (lane == 0) share_sum[item] = ss;
    }
    __syncthreads();
    for (int c = tid * kRun; c < a.hidden; c += step) {
        float v[kRun];
        load_run_f<kRun>(srow + c, v);
        const int g = c / size;                                 // groups are whole runs
        float total = 0.f;
        for (int s = 0; s < shares; ++s) total += share_sum[g * shares + s];
        const float inv = 1.0f / sqrtf(total / static_cast<float>(size) + a.eps);
#pragma unroll
        for (int n = 0; n < kBranchNorms; ++n) {
            if (n >= a.norms) break;
            float gain[kRun];
            load_run_any<kRun>(a.gain[n], c, gain);
            TY* yr = static_cast<TY*>(a.y[n]) + static_cast<long>(blockIdx.x) * a.hidden + c;
            float normed[kRun];
#pragma unroll
            for (int i = 0; i < kRun; ++i) normed[i] = v[i] * inv * gain[i];
            store_run<TY, kRun>(yr, normed);
        }
    }
}

struct StreamJoinArgs {
    float* x;
    BranchTerm term[kBranchTerms];
    int terms;
    const float* first;
    AnyVec next;
    void* operand;
    int hidden;
};

template <typename TY, int kRun>
__global__ void stream_join_kernel(StreamJoinArgs a) {
    const long row = blockIdx.x;
    const int c = (blockIdx.y * blockDim.x + threadIdx.x) * kRun;
    if (c >= a.hidden) return;
    float* xr = a.x + row * a.hidden;
    float v[kRun], f[kRun], n[kRun];
    summed_run<kRun>(xr, a.term, a.terms, row, a.hidden, c, v);
    load_run_f<kRun>(a.first + row * a.hidden + c, f);
    if (a.next.ptr) {
        load_run_any<kRun>(a.next, c, n);
    } else {
#pragma unroll
        for (int i = 0; i < kRun; ++i) n[i] = 0.f;
    }
    TY* to = static_cast<TY*>(a.operand) + row * 2 * a.hidden + c;
    store_run<TY, kRun>(to, v);
    store_run<TY, kRun>(to + a.hidden, f);
    store_run<float, kRun>(xr + c, n);
}

// The results to add, as the entry points take them; whether all of them can be read in runs of four.
static int take_terms(const char* what, BranchTerm* to, const void* const* rows, const int* planes, const long* plane, const float* factor,
                      const void* const* scale, const int* scale_dtype, int terms, bool* runs) {
    LEONE_REQUIRE(terms >= 0 && terms <= kBranchTerms, "%s: %d results, one launch adds at most %d", what, terms, kBranchTerms);
    for (int t = 0; t < terms; ++t) {
        LEONE_REQUIRE(rows[t] && planes[t] >= 1 && planes[t] <= 16 && plane[t] >= 0, "%s: result %d in %d planes", what, t, planes[t]);
        LEONE_REQUIRE(!scale[t] || scale_dtype[t] == kF32 || scale_dtype[t] == kBF16, "%s: unknown type of a scale", what);
        to[t] = BranchTerm{static_cast<const float*>(rows[t]), AnyVec{scale[t], scale_dtype[t]}, factor[t], planes[t], plane[t]};
        *runs = *runs && reinterpret_cast<uintptr_t>(rows[t]) % 16 == 0 && plane[t] % 4 == 0 && reinterpret_cast<uintptr_t>(scale[t]) % 16 == 0;
    }
    return 0;
}

}  // namespace leone

using namespace leone;

// Host arrays of `terms` and `norms` elements; scales may be null one by one.
extern "C" int leone_branch_norm(float* x, const void* const* term_rows, const int* term_planes, const long* term_plane,
                                 const float* term_factor, const void* const* term_scale, const int* term_scale_dtype, int terms,
                                 const void* const* gains, const int* gain_dtypes, void* const* outs, int norms, int out_dtype,
                                 float eps, int groups, const int* rows, int n_rows, int hidden, hipStream_t stream) {
    LEONE_REQUIRE(x && n_rows > 0 && hidden > 0, "branch_norm: rows %d of %d elements", n_rows, hidden);
    LEONE_REQUIRE(terms >= 0 && terms <= kBranchTerms && norms >= 0 && norms <= kBranchNorms && terms + norms > 0,
                  "branch_norm: %d results and %d norms (at most %d and %d)", terms, norms, kBranchTerms, kBranchNorms);
    LEONE_REQUIRE(norms == 0 || (groups > 0 && hidden % groups == 0 && eps > 0.f),
                  "branch_norm: %d elements in %d equal groups, eps %g", hidden, groups, eps);
    LEONE_REQUIRE(out_dtype == kF32 || out_dtype == kBF16, "branch_norm: unknown output type");
    LEONE_REQUIRE(norms > 0 || !rows, "branch_norm: picked rows come with a norm");
    BranchNormArgs a{};
    a.x = x, a.terms = terms, a.norms = norms, a.eps = eps, a.groups = norms ? groups : 1, a.picked = rows, a.hidden = hidden;
    bool runs = hidden % 4 == 0 && (hidden / a.groups) % 4 == 0 && reinterpret_cast<uintptr_t>(x) % 16 == 0;
    if (take_terms("branch_norm", a.term, term_rows, term_planes, term_plane, term_factor, term_scale, term_scale_dtype, terms, &runs)) return 1;
    for (int n = 0; n < norms; ++n) {
        LEONE_REQUIRE(gains[n] && outs[n] && (gain_dtypes[n] == kF32 || gain_dtypes[n] == kBF16), "branch_norm: norm %d needs a gain and room", n);
        a.gain[n] = AnyVec{gains[n], gain_dtypes[n]};
        a.y[n] = outs[n];
        runs = runs && reinterpret_cast<uintptr_t>(gains[n]) % 16 == 0 && reinterpret_cast<uintptr_t>(outs[n]) % 16 == 0;
    }
    // few rows: a row in as few trips to memory as threads allow; many rows: more rows in flight a compute unit
    const int wanted = ceil_div(ceil_div(hidden, runs ? 4 : 1), kWave) * kWave;
    const int most = n_rows < 512 ? kBranchMaxThreads : 256;
    const int threads = wanted < most ? wanted : most;
    const int waves = threads / kWave;
    const int shares = waves / a.groups > 1 ? waves / a.groups : 1;
    const size_t shared = (static_cast<size_t>((hidden + 3) / 4 * 4) + static_cast<size_t>(a.groups) * shares) * sizeof(float);
    LEONE_REQUIRE(shared <= 60 * 1024, "branch_norm: rows of %d elements in %d groups do not fit shared memory", hidden, a.groups);
    if (out_dtype == kBF16) {
        if (runs) branch_norm_kernel<bf16_t, 4><<<n_rows, threads, shared, stream>>>(a);
        else branch_norm_kernel<bf16_t, 1><<<n_rows, threads, shared, stream>>>(a);
    } else {
        if (runs) branch_norm_kernel<float, 4><<<n_rows, threads, shared, stream>>>(a);
        else branch_norm_kernel<float, 1><<<n_rows, threads, shared, stream>>>(a);
    }
    LEONE_LAUNCH_CHECK("branch_norm");
    return 0;
}

// first float [n_rows, hidden]; next [hidden] of next_dtype or null; operand [n_rows, 2 * hidden] of out_dtype.
extern "C" int leone_stream_join(float* x, const void* const* term_rows, const int* term_planes, const long* term_plane,
                                 const float* term_factor, const void* const* term_scale, const int* term_scale_dtype, int terms,
                                 const float* first, const void* next, int next_dtype, void* operand, int out_dtype, int n_rows,
                                 int hidden, hipStream_t stream) {
    LEONE_REQUIRE(x && first && operand && n_rows > 0 && hidden > 0, "stream_join: rows %d of %d elements", n_rows, hidden);
    LEONE_REQUIRE((out_dtype == kF32 || out_dtype == kBF16) && (!next || next_dtype == kF32 || next_dtype == kBF16),
                  "stream_join: unknown element type");
    StreamJoinArgs a{};
    a.x = x, a.terms = terms, a.first = first, a.next = AnyVec{next, next_dtype}, a.operand = operand, a.hidden = hidden;
    bool runs = hidden % 4 == 0 && reinterpret_cast<uintptr_t>(x) % 16 == 0 && reinterpret_cast<uintptr_t>(first) % 16 == 0 &&
                reinterpret_cast<uintptr_t>(next) % 16 == 0 && reinterpret_cast<uintptr_t>(operand) % 16 == 0;
    if (take_terms("stream_join", a.term, term_rows, term_planes, term_plane, term_factor, term_scale, term_scale_dtype, terms, &runs)) return 1;
    const int threads = 256, columns = threads * (runs ? 4 : 1);
    LEONE_REQUIRE(ceil_div(hidden, columns) <= 65535, "stream_join: rows of %d elements", hidden);
    const dim3 grid(n_rows, ceil_div(hidden, columns));
    if (out_dtype == kBF16) {
        if (runs) stream_join_kernel<bf16_t, 4><<<grid, threads, 0, stream>>>(a);
        else stream_join_kernel<bf16_t, 1><<<grid, threads, 0, stream>>>(a);
    } else {
        if (runs) stream_join_kernel<float, 4><<<grid, threads, 0, stream>>>(a);
        else stream_join_kernel<float, 1><<<grid, threads, 0, stream>>>(a);
    }
    LEONE_LAUNCH_CHECK("stream_join");
    return 0;
}
