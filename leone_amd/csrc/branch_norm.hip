// What several sublayers that read the same stream add to it, and the norms that read the stream next, in one kernel:
//
//   branch_norm   x += sum_t factor_t * scale_t * rows_t   (rows_t float [n, hidden], or planes [p, n, hidden] whose sum, in
//                 order, is meant; scale_t a vector [hidden] or absent), then, for up to two norms,
//                 y = x * gain / sqrt(mean over the column's group of x^2 + eps), the columns in `groups` equal groups of
//                 neighbours.  With `picked` only those rows come out and x is left as it was.
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
        load_run_f<kRun>(xr + c, v);
#pragma unroll
        for (int t = 0; t < kBranchTerms; ++t) {
            if (t >= a.terms) break;
            const float* from = a.term[t].rows + in_row * a.hidden + c;
            float d[kRun], s[kRun];
            load_run_f<kRun>(from, d);
            for (int p = 1; p < a.term[t].planes; ++p) {
                float more[kRun];
                load_run_f<kRun>(from + p * a.term[t].plane, more);
#pragma unroll
                for (int i = 0; i < kRun; ++i) d[i] += more[i];
            }
            if (a.term[t].scale.ptr) {
                load_run_any<kRun>(a.term[t].scale, c, s);
#pragma unroll
                for (int i = 0; i < kRun; ++i) v[i] = fmaf(a.term[t].factor * s[i], d[i], v[i]);
            } else {
#pragma unroll
                for (int i = 0; i < kRun; ++i) v[i] = fmaf(a.term[t].factor, d[i], v[i]);
            }
        }
#pragma unroll
        for (int i = 0; i < kRun; ++i) srow[c + i] = v[i];
        if (a.terms > 0 && !a.picked) {
            if constexpr (kRun == 4) {
                *reinterpret_cast<float4*>(xr + c) = float4{v[0], v[1], v[2], v[3]};
            } else {
                xr[c] = v[0];
            }
        }
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
            if constexpr (kRun == 4 && sizeof(TY) == 2) {
                uint2 packed;
                packed.x = bf16_bits_from_float(v[0] * inv * gain[0]) | (static_cast<uint32_t>(bf16_bits_from_float(v[1] * inv * gain[1])) << 16);
                packed.y = bf16_bits_from_float(v[2] * inv * gain[2]) | (static_cast<uint32_t>(bf16_bits_from_float(v[3] * inv * gain[3])) << 16);
                *reinterpret_cast<uint2*>(yr) = packed;
            } else {
#pragma unroll
                for (int i = 0; i < kRun; ++i) yr[i] = from_float<TY>(v[i] * inv * gain[i]);
            }
        }
    }
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
    for (int t = 0; t < terms; ++t) {
        LEONE_REQUIRE(term_rows[t] && term_planes[t] >= 1 && term_planes[t] <= 16 && term_plane[t] >= 0,
                      "branch_norm: result %d in %d planes", t, term_planes[t]);
        LEONE_REQUIRE(!term_scale[t] || term_scale_dtype[t] == kF32 || term_scale_dtype[t] == kBF16, "branch_norm: unknown type of a scale");
        a.term[t] = BranchTerm{static_cast<const float*>(term_rows[t]), AnyVec{term_scale[t], term_scale_dtype[t]}, term_factor[t],
                               term_planes[t], term_plane[t]};
        runs = runs && reinterpret_cast<uintptr_t>(term_rows[t]) % 16 == 0 && term_plane[t] % 4 == 0 &&
               reinterpret_cast<uintptr_t>(term_scale[t]) % 16 == 0;
    }
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
