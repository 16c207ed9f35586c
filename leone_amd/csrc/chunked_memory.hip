// Matrix memories with one decay a head, over long portions, as products on the matrix cores (float throughout).
//
//   S_t = g_t S_(t-1) + k_t u_t^T,  o_t = S_t^T q_t                                       S is [dim, vdim]
//   fixed decays:   g a constant of the head, u_t = v_t
//   delta rule:     u_t = beta_t (v_t - (g_t S_(t-1))^T k_t)
//
// Over a chunk of 64 rows, with L_t the product of the chunk's decays up to and with row t and S0 the state it starts from,
//   S_t = L_t S0 + sum_(i <= t) (L_t / L_i) k_i u_i^T,
// so with A_ti = beta_t (L_t / L_i) k_t.k_i (i < t) and M_ti = (L_t / L_i) q_t.k_i (i <= t), one row a token,
//   (1 + A) U = diag(beta) V - diag(beta L) K S0,   O = diag(L) Q S0 + M U,   S_end = L_end S0 + (diag(L_end / L) K)^T U.
// chunk_prepare makes everything that does not hold S0, all chunks and heads side by side: U0 and W, the solutions of the
// triangular system for diag(beta) V and diag(beta L) K (forward substitution, 16 rows at a time: the rows before leave them
// as products), M, and Q and K with their decays.  chunk_walk then goes through a portion's chunks in order, a workgroup a head
// and 16 columns of S: U = U0 - W S, O, S.  With fixed decays there is no system: U = V.
//
// Products are v_mfma_f32_16x16x4_f32.  Lane l = 16 g + c holds A[row c][k-slot g], B[k-slot g][column c] and rows 4 g + v of
// column c of the result in register v.  Which inner element a k-slot stands for is free as long as both operands agree:
// instruction v of a run of 16 takes element 4 g + v for slot g, so that an operand is one 16-byte read a lane, and a result
// in registers (S, U) is the next product's second operand as it lies.  Decays travel as logarithms summed over the chunk, in
// double: a row that forgets everything must not blur the small decays behind it.
#include "common.h"
#include "leone_hip.h"

#include <math.h>

namespace leone {

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;

constexpr int kChunkRows = 64;
constexpr int kChunkThreads = 256;
constexpr int kChunkMaxDim = 128;       // key channels: two tiles of 16 a wave
constexpr int kChunkTiles = 10;         // tiles of 16 x 16 of a chunk's rows by rows on and below the diagonal
constexpr int kPartStride = 20;         // of a row of 16 in shared memory: rows four apart lie in banks of their own

struct ChunkArgs {
    const float* rows;          // [rows, stride]: q and k heads (kv_heads x dim each), v heads (heads x vdim)
    long stride;
    int q_off, k_off, v_off;
    int silu;                   // q, k and v pass through silu first
    float q_scale, k_scale;
    float unit_eps;             // delta rule: q and k are made unit vectors a head first, this under the root
    const float* beta;          // delta rule: [rows, beta_stride] pre-activation of the write strength, one a head
    long beta_stride;
    const float* step;          // delta rule: [rows, step_stride] pre-activation of the step size, one a head
    long step_stride;
    AnyVec rate_log, step_bias; // delta rule: [heads]; decay = exp(-exp(rate_log) * softplus(step + step_bias))
    const float* decay;         // fixed decays: [heads]
    const int* chunks;          // [chunks, 4]: first row, end, -, -
    const int* links;           // [links, 4]: state slot, whether the sequence starts here, first chunk, end
    float* q_in;                // [chunks, heads, 64 x dim_p]: q_t L_t, in the order chunk_walk reads
    float* k_out;               // [chunks, heads, dim_p x 64]: k_t L_end / L_t, likewise
    float* mix;                 // [chunks, heads, 64 x 64]: M, likewise (tiles above the diagonal are not written)
    float* solved_k;            // delta rule: [chunks, heads, 64 x dim_p]: W, likewise
    float* values;              // [chunks, heads, 64, vdim_p]: U0, or V
    float* total;               // [chunks, heads]: L_end
    float* state;               // [slots, heads, dim, vdim]
    long slot_stride;
    int write_state;
    float* out;                 // [rows, heads, vdim]
    int heads, kv_heads, dim, vdim, dim_p, vdim_p;      // _p: filled up to whole tiles
};

__device__ inline float chunk_act(float x, int silu) { return silu ? x / (1.0f + expf(-x)) : x; }
__device__ inline float chunk_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }
constexpr float kNothingLeft = -1e4f;   // a logarithm whose exponential is zero and of which 64 add up without overflow
__device__ inline float between(double later, double earlier) { return expf(static_cast<float>(later - earlier)); }
__device__ inline floatx4 mfma4(float a, float b, floatx4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// Where the four elements that a lane of chunk_walk reads at once stand in the chunk's rows: its operands lie in the order of
// [wave][tile of rows][tile of channels][lane], so that a wave reads 1,024 bytes in a row.
struct Place { int row, channel; };
template <int kT>
__device__ inline Place place_of(int idx) {
    const int lane = idx % kWave, tile = idx / kWave;
    return {16 * (tile / kT % 4) + (lane & 15), 16 * (tile / (4 * kT) * kT + tile % kT) + 4 * (lane >> 4)};
}

// kT: tiles of 16 key channels a wave of chunk_walk holds; 64 kT channels, the last ones zeros.
template <bool kDelta, int kT>
__global__ void __launch_bounds__(kChunkThreads, 2) chunk_prepare_kernel(ChunkArgs p) {
    extern __shared__ __align__(16) float chunk_lds[];
    constexpr int kDim = 64 * kT, row_p = kDim + 4;
    float* sq = chunk_lds;                              // [64][row_p]
    float* sk = sq + kChunkRows * row_p;
    float* sa = sk + kChunkRows * row_p;                // delta rule: -A in tiles of 16 x 16, those on and below the diagonal
    __shared__ double cum[kChunkRows];
    __shared__ float strength[kChunkRows], q_norm[kChunkRows], k_norm[kChunkRows], so_far[kChunkRows], to_end[kChunkRows];
    const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
    const int chunk = blockIdx.x, head = blockIdx.y, kvh = head / (p.heads / p.kv_heads);
    const int first = p.chunks[4 * chunk], n = p.chunks[4 * chunk + 1] - first;
    const long at = static_cast<long>(chunk) * p.heads + head;
    const int block = blockIdx.z * kDim;        // delta rule: the value columns solved here; the first workgroup writes all the rest

    // reads in batches, of the last row or channel again where there is none, so that no read waits for the one before
    constexpr int kBatch = 8;
    static_assert(kChunkRows * kDim % (kBatch * kChunkThreads) == 0, "whole batches");
    for (int from = tid; from < kChunkRows * kDim; from += kBatch * kChunkThreads) {
        float q[kBatch], k[kBatch];
#pragma unroll
        for (int e = 0; e < kBatch; ++e) {
            const int t = (from + e * kChunkThreads) / kDim, i = (from + e * kChunkThreads) % kDim;
            const float* base = p.rows + static_cast<long>(first + min(t, n - 1)) * p.stride + kvh * p.dim + min(i, p.dim - 1);
            q[e] = base[p.q_off], k[e] = base[p.k_off];
        }
#pragma unroll
        for (int e = 0; e < kBatch; ++e) {
            const int t = (from + e * kChunkThreads) / kDim, i = (from + e * kChunkThreads) % kDim;
            const bool there = t < n && i < p.dim;
            sq[t * row_p + i] = there ? chunk_act(q[e], p.silu) : 0.f;
            sk[t * row_p + i] = there ? chunk_act(k[e], p.silu) : 0.f;
        }
    }
    if (wave == 0) {
        // the decays' logarithms summed up over the chunk; rows past its end decay nothing and write nothing
        double l = 0.;
        if (lane < n) {
            const long row = first + lane;
            if (kDelta) {
                l = -expf(load_any(p.rate_log, head)) * chunk_softplus(p.step[row * p.step_stride + head] + load_any(p.step_bias, head));
                strength[lane] = 1.0f / (1.0f + expf(-p.beta[row * p.beta_stride + head]));
            } else {
                const float d = p.decay[head];
                l = d > 0.f ? logf(d) : kNothingLeft;
            }
            l = fmax(l, static_cast<double>(kNothingLeft));
        } else if (kDelta) {
            strength[lane] = 0.f;
        }
#pragma unroll
        for (int off = 1; off < kWave; off <<= 1) {
            const double before = __shfl_up(l, off, kWave);
            if (lane >= off) l += before;
        }
        cum[lane] = l;
        so_far[lane] = between(l, 0.);
        to_end[lane] = between(__shfl(l, kWave - 1, kWave), l);
    }
    __syncthreads();
    {   // four lanes a row
        const int t = tid / 4, sub = tid % 4;
        float qq = 0.f, kk = 0.f;
        if (kDelta) {
            for (int i = sub; i < p.dim; i += 4) {
                qq = fmaf(sq[t * row_p + i], sq[t * row_p + i], qq);
                kk = fmaf(sk[t * row_p + i], sk[t * row_p + i], kk);
            }
            qq += __shfl_xor(qq, 1, kWave);
            kk += __shfl_xor(kk, 1, kWave);
            qq += __shfl_xor(qq, 2, kWave);
            kk += __shfl_xor(kk, 2, kWave);
        }
        if (sub == 0) {
            q_norm[t] = kDelta ? p.q_scale / sqrtf(qq + p.unit_eps) : p.q_scale;
            k_norm[t] = kDelta ? p.k_scale / sqrtf(kk + p.unit_eps) : p.k_scale;
        }
    }
    __syncthreads();
    if (tid == 0 && block == 0) p.total[at] = so_far[kChunkRows - 1];

    // k_t.k_i and q_t.k_i, the ten tiles of 16 x 16 on and below the diagonal shared out over the waves
    float* mix = p.mix + at * kChunkRows * kChunkRows;
    const int c = lane & 15, g = lane >> 4;
    for (int pair = wave; pair < kChunkTiles; pair += kChunkThreads / kWave) {
        const int ti = pair < 1 ? 0 : pair < 3 ? 1 : pair < 6 ? 2 : 3, tj = pair - ti * (ti + 1) / 2;
        const float* rq = sq + (16 * ti + c) * row_p + 4 * g;
        const float* rk = sk + (16 * ti + c) * row_p + 4 * g;
        const float* ck = sk + (16 * tj + c) * row_p + 4 * g;
        floatx4 kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int d = 0; d < kDim; d += 16) {
            const float4 b = *reinterpret_cast<const float4*>(ck + d), aq = *reinterpret_cast<const float4*>(rq + d);
            qk = mfma4(aq.x, b.x, qk);
            qk = mfma4(aq.y, b.y, qk);
            qk = mfma4(aq.z, b.z, qk);
            qk = mfma4(aq.w, b.w, qk);
            if (kDelta) {
                const float4 ak = *reinterpret_cast<const float4*>(rk + d);
                kk = mfma4(ak.x, b.x, kk);
                kk = mfma4(ak.y, b.y, kk);
                kk = mfma4(ak.z, b.z, kk);
                kk = mfma4(ak.w, b.w, kk);
            }
        }
        const int i = 16 * tj + c;
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const int t = 16 * ti + 4 * g + v;
            const float decayed = t >= i ? between(cum[t], cum[i]) * k_norm[i] : 0.f;
            if (block == 0) mix[4 * ((ti * 4 + tj) * kWave + 16 * (c / 4) + 4 * g + v) + c % 4] = decayed * q_norm[t] * qk[v];
            if (kDelta) sa[256 * pair + 16 * (4 * g + v) + c] = -decayed * k_norm[t] * strength[t] * kk[v];
        }
    }
    float* q_in = p.q_in + at * kChunkRows * kDim;
    float* k_out = p.k_out + at * kChunkRows * kDim;
    if (block == 0) {
#pragma unroll 4
        for (int idx = tid; idx < kChunkRows * kDim / 4; idx += kChunkThreads) {
            const Place a = place_of<kT>(idx);
            const float4 x = *reinterpret_cast<const float4*>(sq + a.row * row_p + a.channel);
            const float f = q_norm[a.row] * so_far[a.row];
            reinterpret_cast<float4*>(q_in)[idx] = float4{x.x * f, x.y * f, x.z * f, x.w * f};
            const int ki = 16 * (idx / kWave / 4) + c, kt = 16 * (idx / kWave % 4) + 4 * g;
            float4 y;
            y.x = sk[kt * row_p + ki] * (k_norm[kt] * to_end[kt]);
            y.y = sk[(kt + 1) * row_p + ki] * (k_norm[kt + 1] * to_end[kt + 1]);
            y.z = sk[(kt + 2) * row_p + ki] * (k_norm[kt + 2] * to_end[kt + 2]);
            y.w = sk[(kt + 3) * row_p + ki] * (k_norm[kt + 3] * to_end[kt + 3]);
            reinterpret_cast<float4*>(k_out)[idx] = y;
        }
    }
    float* values = p.values + at * kChunkRows * p.vdim_p;
    const float* v_base = p.rows + static_cast<long>(first) * p.stride + p.v_off + head * p.vdim;
    const auto read_v = [&](int t, int j) { return v_base[min(t, n - 1) * p.stride + min(j, p.vdim - 1)]; };
    const auto taken_v = [&](float v, int t, int j) { return t < n && j < p.vdim ? chunk_act(v, p.silu) : 0.f; };
    if constexpr (!kDelta) {
        constexpr int kRows = kChunkThreads / kWave, kEach = kChunkRows / kRows;
        for (int j = lane; j < p.vdim_p; j += kWave) {
            float v[kEach];
#pragma unroll
            for (int e = 0; e < kEach; ++e) v[e] = read_v(wave + kRows * e, j);
#pragma unroll
            for (int e = 0; e < kEach; ++e) values[(wave + kRows * e) * p.vdim_p + j] = taken_v(v[e], wave + kRows * e, j);
        }
    } else {
        float* solved_k = p.solved_k + at * kChunkRows * kDim;
        __syncthreads();                    // M is made and K written: their places take the right sides, K and a block of V
        for (int from = tid; from < kChunkRows * kDim; from += kBatch * kChunkThreads) {
            float v[kBatch];
#pragma unroll
            for (int e = 0; e < kBatch; ++e) v[e] = read_v((from + e * kChunkThreads) / kDim, block + (from + e * kChunkThreads) % kDim);
#pragma unroll
            for (int e = 0; e < kBatch; ++e) {
                const int t = (from + e * kChunkThreads) / kDim, i = (from + e * kChunkThreads) % kDim;
                sk[t * row_p + i] *= strength[t] * so_far[t] * k_norm[t];
                sq[t * row_p + i] = strength[t] * taken_v(v[e], t, block + i);
            }
        }
        __syncthreads();
        static_assert(2 * kDim <= kChunkThreads, "a thread takes one column");
        const bool is_key = tid >= kDim;
        const int mine = is_key ? tid - kDim : tid;
        float* column = (is_key ? sk : sq) + mine;
        float* to = values + block + mine;
        const bool stores = !is_key && block + mine < p.vdim_p;
#pragma unroll 1
        for (int b = 0; b < kChunkRows / 16; ++b) {
            // 16 rows at a time: the solved rows leave them as products,
            const float* tiles = sa + 256 * (b * (b + 1) / 2);
            if (b > 0) {
                for (int at16 = wave; at16 < 2 * kDim / 16; at16 += kChunkThreads / kWave) {
                    float* x = (at16 < kDim / 16 ? sq + 16 * at16 : sk + 16 * at16 - kDim) + c;
                    floatx4 sum;
#pragma unroll
                    for (int v = 0; v < 4; ++v) sum[v] = x[(16 * b + 4 * g + v) * row_p];
                    for (int s = 0; s < b; ++s) {
                        const float4 a = *reinterpret_cast<const float4*>(tiles + 256 * s + 16 * c + 4 * g);
                        const float* solved = x + (16 * s + 4 * g) * row_p;
                        sum = mfma4(a.x, solved[0], sum);
                        sum = mfma4(a.y, solved[row_p], sum);
                        sum = mfma4(a.z, solved[2 * row_p], sum);
                        sum = mfma4(a.w, solved[3 * row_p], sum);
                    }
#pragma unroll
                    for (int v = 0; v < 4; ++v) x[(16 * b + 4 * g + v) * row_p] = sum[v];
                }
                __syncthreads();
            }
            // then a column a thread among themselves
            if (tid < 2 * kDim) {
                float x[16];
#pragma unroll
                for (int t = 0; t < 16; ++t) x[t] = column[(16 * b + t) * row_p];
#pragma unroll
                for (int t = 1; t < 16; ++t)
#pragma unroll
                    for (int i4 = 0; 4 * i4 < t; ++i4) {
                        const float4 a = *reinterpret_cast<const float4*>(tiles + 256 * b + 16 * t + 4 * i4);
                        x[t] = fmaf(a.x, x[4 * i4], x[t]);
                        if (4 * i4 + 1 < t) x[t] = fmaf(a.y, x[4 * i4 + 1], x[t]);
                        if (4 * i4 + 2 < t) x[t] = fmaf(a.z, x[4 * i4 + 2], x[t]);
                        if (4 * i4 + 3 < t) x[t] = fmaf(a.w, x[4 * i4 + 3], x[t]);
                    }
#pragma unroll
                for (int t = 0; t < 16; ++t) {
                    column[(16 * b + t) * row_p] = x[t];
                    if (stores) to[(16 * b + t) * p.vdim_p] = x[t];
                }
            }
            __syncthreads();
        }
        if (block == 0)
#pragma unroll 4
            for (int idx = tid; idx < kChunkRows * kDim / 4; idx += kChunkThreads) {
                const Place a = place_of<kT>(idx);
                reinterpret_cast<float4*>(solved_k)[idx] = *reinterpret_cast<const float4*>(sk + a.row * row_p + a.channel);
            }
    }
}

// What a wave needs of a chunk, all of it asked for a chunk ahead.
template <bool kDelta, int kT>
struct ChunkOperands {
    float4 w[kDelta ? 4 : 1][kT], q[4][kT], k[kT][4], m[4];
    float u[4], total;
    int first, end;
};

template <bool kDelta, int kT>
__device__ inline void fetch_chunk(const ChunkArgs& p, int chunk, int head, int wave, int c, int g, int col, ChunkOperands<kDelta, kT>& o) {
    const long at = static_cast<long>(chunk) * p.heads + head;
    constexpr int kDim = 64 * kT;
    const int lane = 16 * g + c;
    const float4* q_in = reinterpret_cast<const float4*>(p.q_in + at * kChunkRows * kDim) + wave * 4 * kT * kWave + lane;
    const float4* k_out = reinterpret_cast<const float4*>(p.k_out + at * kChunkRows * kDim) + wave * 4 * kT * kWave + lane;
    const float4* mix = reinterpret_cast<const float4*>(p.mix + at * kChunkRows * kChunkRows) + wave * 4 * kWave + lane;
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int t = 0; t < kT; ++t) {
            if constexpr (kDelta)
                o.w[r][t] = (reinterpret_cast<const float4*>(p.solved_k + at * kChunkRows * kDim) + wave * 4 * kT * kWave + lane)[(r * kT + t) * kWave];
            o.q[r][t] = q_in[(r * kT + t) * kWave];
        }
    o.first = p.chunks[4 * chunk];
    o.end = p.chunks[4 * chunk + 1];
    o.total = p.total[at];
#pragma unroll
    for (int v = 0; v < 4; ++v) o.u[v] = p.values[at * kChunkRows * p.vdim_p + (16 * wave + 4 * g + v) * p.vdim_p + col];
#pragma unroll
    for (int s = 0; s < 4; ++s) o.m[s] = s <= wave ? mix[s * kWave] : float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < kT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) o.k[t][r] = k_out[(t * 4 + r) * kWave];
}

__device__ inline float element(const float4& f, int v) { return v == 0 ? f.x : v == 1 ? f.y : v == 2 ? f.z : f.w; }

// A workgroup walks the chunks of one portion for one head and 16 columns; wave w holds key channels 16 kT w .. of the columns
// and makes what they give to every row of W S and Q S; the parts meet in shared memory, where wave w takes rows 16 w ..
template <bool kDelta, int kT>
__global__ void __launch_bounds__(kChunkThreads, 1) chunk_walk_kernel(ChunkArgs p) {
    constexpr int kWaves = kChunkThreads / kWave;
    __shared__ float part[kDelta ? 2 : 1][kWaves][kChunkRows * kPartStride];
    __shared__ float su[kChunkRows * kPartStride];
    const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, c = lane & 15, g = lane >> 4;
    const int link = blockIdx.x, head = blockIdx.y, col = 16 * blockIdx.z + c;
    const int slot = p.links[4 * link], fresh = p.links[4 * link + 1], g0 = p.links[4 * link + 2], g1 = p.links[4 * link + 3];
    float* state = p.state + slot * p.slot_stride + static_cast<long>(head) * p.dim * p.vdim;
    floatx4 S[kT];
#pragma unroll
    for (int t = 0; t < kT; ++t)
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const int i = 16 * (wave * kT + t) + 4 * g + v;
            S[t][v] = (!fresh && i < p.dim && col < p.vdim) ? state[static_cast<long>(i) * p.vdim + col] : 0.f;
        }
    if (g0 >= g1) return;
    ChunkOperands<kDelta, kT> ahead;
    fetch_chunk<kDelta, kT>(p, g0, head, wave, c, g, col, ahead);
    for (int chunk = g0; chunk < g1; ++chunk) {
        const ChunkOperands<kDelta, kT> now = ahead;
        fetch_chunk<kDelta, kT>(p, chunk + 1 < g1 ? chunk + 1 : chunk, head, wave, c, g, col, ahead);
        floatx4 ws[4], qs[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) ws[r] = qs[r] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < kT; ++t)
#pragma unroll
            for (int v = 0; v < 4; ++v)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    if constexpr (kDelta) ws[r] = mfma4(element(now.w[r][t], v), S[t][v], ws[r]);
                    qs[r] = mfma4(element(now.q[r][t], v), S[t][v], qs[r]);
                }
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
            for (int v = 0; v < 4; ++v) {
                part[0][wave][(16 * r + 4 * g + v) * kPartStride + c] = qs[r][v];
                if constexpr (kDelta) part[kDelta ? 1 : 0][wave][(16 * r + 4 * g + v) * kPartStride + c] = ws[r][v];
            }
        __syncthreads();
        floatx4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const int place = (16 * wave + 4 * g + v) * kPartStride + c;
            float seen = 0.f;
#pragma unroll
            for (int w = 0; w < kWaves; ++w) {
                o[v] += part[0][w][place];
                if constexpr (kDelta) seen += part[kDelta ? 1 : 0][w][place];
            }
            su[place] = now.u[v] - seen;
        }
        __syncthreads();
        float u[4][4];
#pragma unroll
        for (int s = 0; s < 4; ++s)
#pragma unroll
            for (int v = 0; v < 4; ++v) u[s][v] = su[(16 * s + 4 * g + v) * kPartStride + c];
#pragma unroll
        for (int t = 0; t < kT; ++t) S[t] *= now.total;
#pragma unroll
        for (int s = 0; s < 4; ++s)
#pragma unroll
            for (int v = 0; v < 4; ++v) {
                o = mfma4(element(now.m[s], v), u[s][v], o);            // tiles above the diagonal are zeros
#pragma unroll
                for (int t = 0; t < kT; ++t) S[t] = mfma4(element(now.k[t][s], v), u[s][v], S[t]);
            }
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const int t = 16 * wave + 4 * g + v;
            if (now.first + t < now.end && col < p.vdim) p.out[(static_cast<long>(now.first + t) * p.heads + head) * p.vdim + col] = o[v];
        }
    }
    if (!p.write_state) return;
#pragma unroll
    for (int t = 0; t < kT; ++t)
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const int i = 16 * (wave * kT + t) + 4 * g + v;
            if (i < p.dim && col < p.vdim) state[static_cast<long>(i) * p.vdim + col] = S[t][v];
        }
}

static int chunk_tiles(int dim) { return dim <= 64 ? 1 : 2; }      // tiles of 16 key channels a wave

}  // namespace leone

using namespace leone;

extern "C" int leone_chunk_rows() { return kChunkRows; }
extern "C" int leone_chunk_max_dim() { return kChunkMaxDim; }

// Floats of workspace a chunk and head needs; delta: the delta rule.
extern "C" long leone_chunk_workspace(int dim, int vdim, int delta) {
    const long dim_p = 64L * chunk_tiles(dim), vdim_p = ceil_div(vdim, 16) * 16L;
    return kChunkRows * (dim_p * (delta ? 3 : 2) + vdim_p + kChunkRows) + 4;
}

// A long portion's rows through a memory with one decay a head.  beta, step, rate_log and step_bias belong to the delta rule
// (all null: fixed decays from `decay`); the delta rule makes q and k unit vectors first.  chunks and links: the portions' chunks
// of leone_chunk_rows() rows as the other recurrences list them.  workspace: n_chunks * heads * leone_chunk_workspace() floats.
extern "C" int leone_chunked_memory(const float* rows, long stride, int q_off, int k_off, int v_off, int silu, float q_scale,
                                    float k_scale, float unit_eps, const float* beta, long beta_stride, const float* step,
                                    long step_stride, const void* rate_log, const void* step_bias, int vec_dtype,
                                    const float* decay, const int* chunks, int n_chunks, const int* links, int n_links,
                                    float* workspace, float* state, long slot_stride, int write_state, float* out, int heads,
                                    int kv_heads, int dim, int vdim, hipStream_t stream) {
    const bool delta = beta != nullptr;
    LEONE_REQUIRE(rows && chunks && links && workspace && state && out && n_chunks > 0 && n_links > 0, "chunked_memory: null pointer or no chunks");
    LEONE_REQUIRE(delta ? (step && rate_log && step_bias && unit_eps > 0.f && (vec_dtype == kF32 || vec_dtype == kBF16)) : decay != nullptr,
                  "chunked_memory: the delta rule needs strengths, step sizes and rates, anything else fixed decays");
    LEONE_REQUIRE(heads > 0 && heads <= 65535 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && dim <= kChunkMaxDim && vdim > 0 && vdim <= 16 * 65535,
                  "chunked_memory: %d heads over %d key heads of %d x %d (at most %d key channels)", heads, kv_heads, dim, vdim, kChunkMaxDim);
    LEONE_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && stride >= q_off + static_cast<long>(kv_heads) * dim &&
                  stride >= k_off + static_cast<long>(kv_heads) * dim && stride >= v_off + static_cast<long>(heads) * vdim &&
                  (!delta || (beta_stride >= heads && step_stride >= heads)), "chunked_memory: rows of %ld do not hold the named columns", stride);
    LEONE_REQUIRE(slot_stride >= static_cast<long>(heads) * dim * vdim, "chunked_memory: states of %ld floats do not fit", slot_stride);
    LEONE_REQUIRE(reinterpret_cast<uintptr_t>(workspace) % 16 == 0, "chunked_memory: the workspace must be aligned to 16 bytes");
    ChunkArgs a{};
    a.rows = rows, a.stride = stride, a.q_off = q_off, a.k_off = k_off, a.v_off = v_off, a.silu = silu;
    a.q_scale = q_scale, a.k_scale = k_scale, a.unit_eps = unit_eps;
    a.beta = beta, a.beta_stride = beta_stride, a.step = step, a.step_stride = step_stride;
    a.rate_log = AnyVec{rate_log, vec_dtype}, a.step_bias = AnyVec{step_bias, vec_dtype}, a.decay = decay;
    a.chunks = chunks, a.links = links, a.state = state, a.slot_stride = slot_stride, a.write_state = write_state, a.out = out;
    a.heads = heads, a.kv_heads = kv_heads, a.dim = dim, a.vdim = vdim;
    const int tiles = chunk_tiles(dim);
    a.dim_p = 64 * tiles, a.vdim_p = ceil_div(vdim, 16) * 16;
    const long each = static_cast<long>(n_chunks) * heads * kChunkRows;
    a.q_in = workspace;
    a.k_out = a.q_in + each * a.dim_p;
    a.values = a.k_out + each * a.dim_p;
    a.mix = a.values + each * a.vdim_p;
    a.solved_k = a.mix + each * kChunkRows;
    a.total = a.solved_k + (delta ? each * a.dim_p : 0);
    const size_t shared = (2 * kChunkRows * (a.dim_p + 4) + (delta ? kChunkTiles * 256 : 0)) * sizeof(float);
    static bool allowed = false;
    if (!allowed) {
        const int most = (2 * kChunkRows * (kChunkMaxDim + 4) + kChunkTiles * 256) * sizeof(float);
        for (const void* kernel : {reinterpret_cast<const void*>(&chunk_prepare_kernel<false, 1>), reinterpret_cast<const void*>(&chunk_prepare_kernel<false, 2>),
                                   reinterpret_cast<const void*>(&chunk_prepare_kernel<true, 1>), reinterpret_cast<const void*>(&chunk_prepare_kernel<true, 2>)}) {
            const hipError_t e = hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, most);
            LEONE_REQUIRE(e == hipSuccess, "chunked_memory: %d bytes of shared memory were refused: %s", most, hipGetErrorString(e));
        }
        allowed = true;
    }
    const dim3 prepare(n_chunks, heads, delta ? ceil_div(a.vdim_p, a.dim_p) : 1), walk(n_links, heads, a.vdim_p / 16);
    if (delta) {
        if (tiles == 1) chunk_prepare_kernel<true, 1><<<prepare, kChunkThreads, shared, stream>>>(a);
        else chunk_prepare_kernel<true, 2><<<prepare, kChunkThreads, shared, stream>>>(a);
        LEONE_LAUNCH_CHECK("chunk_prepare");
        if (tiles == 1) chunk_walk_kernel<true, 1><<<walk, kChunkThreads, 0, stream>>>(a);
        else chunk_walk_kernel<true, 2><<<walk, kChunkThreads, 0, stream>>>(a);
    } else {
        if (tiles == 1) chunk_prepare_kernel<false, 1><<<prepare, kChunkThreads, shared, stream>>>(a);
        else chunk_prepare_kernel<false, 2><<<prepare, kChunkThreads, shared, stream>>>(a);
        LEONE_LAUNCH_CHECK("chunk_prepare");
        if (tiles == 1) chunk_walk_kernel<false, 1><<<walk, kChunkThreads, 0, stream>>>(a);
        else chunk_walk_kernel<false, 2><<<walk, kChunkThreads, 0, stream>>>(a);
    }
    LEONE_LAUNCH_CHECK("chunk_walk");
    return 0;
}
