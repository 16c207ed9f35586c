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
// triangular system for diag(beta) V and diag(beta L) K (forward substitution, a column a thread, the chunk's 64 values of a
// column in registers), M, and Q and K with their decays.  chunk_walk then goes through a portion's chunks in order, a
// workgroup a head and 16 columns of S: U = U0 - W S, O, S.  With fixed decays there is no system: U = V.
//
// Products are v_mfma_f32_16x16x4_f32.  Lane l = 16 g + c holds A[row c][k-slot g], B[k-slot g][column c] and rows 4 g + v of
// column c of the result in register v.  Which inner element a k-slot stands for is free as long as both operands agree:
// instruction v of a run of 16 takes element 4 g + v for slot g, so that an operand is one 16-byte read a lane, and a result
// in registers (S, U) is the next product's second operand as it lies.  Decays travel as logarithms summed over the chunk, in double:
// a row that forgets everything must not blur the small decays behind it.
#include "common.h"
#include "leone_hip.h"

#include <math.h>

namespace leone {

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;

constexpr int kChunkRows = 64;
constexpr int kChunkThreads = 256;
constexpr int kChunkMaxDim = 128;       // key channels: two tiles of 16 a wave
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
    float* q_in;                // [chunks, heads, 64, dim_p]: q_t L_t
    float* k_out;               // [chunks, heads, dim_p, 64]: k_t L_end / L_t
    float* mix;                 // [chunks, heads, 64, 64]: M (tiles above the diagonal are not written)
    float* solved_k;            // delta rule: [chunks, heads, 64, dim_p]: W
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

template <bool kDelta>
__global__ void __launch_bounds__(kChunkThreads, 1) chunk_prepare_kernel(ChunkArgs p) {
    extern __shared__ __align__(16) float chunk_lds[];
    const int row_p = p.dim_p + 4;
    float* sq = chunk_lds;                              // [64][row_p]
    float* sk = sq + kChunkRows * row_p;
    float* sa = sk + kChunkRows * row_p;                // [64][68]: A turned, column i of A at row i (delta rule only)
    constexpr int kAStride = kChunkRows + 4;
    __shared__ double cum[kChunkRows];
    __shared__ float strength[kChunkRows], q_norm[kChunkRows], k_norm[kChunkRows];
    const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
    const int chunk = blockIdx.x, head = blockIdx.y, kvh = head / (p.heads / p.kv_heads);
    const int first = p.chunks[4 * chunk], n = p.chunks[4 * chunk + 1] - first;
    const long at = static_cast<long>(chunk) * p.heads + head;

    for (int idx = tid; idx < kChunkRows * p.dim_p; idx += kChunkThreads) {
        const int t = idx / p.dim_p, i = idx % p.dim_p;
        float q = 0.f, k = 0.f;
        if (t < n && i < p.dim) {
            const float* base = p.rows + static_cast<long>(first + t) * p.stride + kvh * p.dim + i;
            q = chunk_act(base[p.q_off], p.silu);
            k = chunk_act(base[p.k_off], p.silu);
        }
        sq[t * row_p + i] = q;
        sk[t * row_p + i] = k;
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
    if (tid == 0) p.total[at] = between(cum[kChunkRows - 1], 0.);

    // k_t.k_i and q_t.k_i, the ten tiles of 16 x 16 on and below the diagonal shared out over the waves
    float* mix = p.mix + at * kChunkRows * kChunkRows;
    const int c = lane & 15, g = lane >> 4;
    for (int pair = wave; pair < 10; pair += kChunkThreads / kWave) {
        const int ti = pair < 1 ? 0 : pair < 3 ? 1 : pair < 6 ? 2 : 3, tj = pair - ti * (ti + 1) / 2;
        const float* rq = sq + (16 * ti + c) * row_p + 4 * g;
        const float* rk = sk + (16 * ti + c) * row_p + 4 * g;
        const float* ck = sk + (16 * tj + c) * row_p + 4 * g;
        floatx4 kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};
        for (int d = 0; d < p.dim_p; d += 16) {
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
            mix[t * kChunkRows + i] = decayed * q_norm[t] * qk[v];
            if (kDelta) sa[i * kAStride + t] = decayed * k_norm[t] * strength[t] * kk[v];
        }
    }
    float* q_in = p.q_in + at * kChunkRows * p.dim_p;
    float* k_out = p.k_out + at * kChunkRows * p.dim_p;
    for (int idx = tid; idx < kChunkRows * p.dim_p; idx += kChunkThreads) {
        const int t = idx / p.dim_p, i = idx % p.dim_p;
        q_in[idx] = sq[t * row_p + i] * q_norm[t] * between(cum[t], 0.);
        const int kt = idx % kChunkRows, ki = idx / kChunkRows;
        k_out[idx] = sk[kt * row_p + ki] * k_norm[kt] * between(cum[kChunkRows - 1], cum[kt]);
    }
    float* values = p.values + at * kChunkRows * p.vdim_p;
    const float* v_base = p.rows + static_cast<long>(first) * p.stride + p.v_off + head * p.vdim;
    if constexpr (!kDelta) {
        for (int idx = tid; idx < kChunkRows * p.vdim_p; idx += kChunkThreads) {
            const int t = idx / p.vdim_p, j = idx % p.vdim_p;
            values[idx] = (t < n && j < p.vdim) ? chunk_act(v_base[t * p.stride + j], p.silu) : 0.f;
        }
    } else {
        __syncthreads();
        float* solved_k = p.solved_k + at * kChunkRows * p.dim_p;
        for (int col = tid; col < p.dim_p + p.vdim_p; col += kChunkThreads) {
            const bool is_key = col < p.dim_p;
            const int j = is_key ? col : col - p.dim_p;
            float x[kChunkRows];
#pragma unroll
            for (int t = 0; t < kChunkRows; ++t) {
                if (is_key) x[t] = strength[t] * between(cum[t], 0.) * k_norm[t] * sk[t * row_p + j];
                else x[t] = (t < n && j < p.vdim) ? strength[t] * chunk_act(v_base[t * p.stride + j], p.silu) : 0.f;
            }
#pragma unroll
            for (int i = 0; i < kChunkRows - 1; ++i) {
                // row i is solved: it leaves every row behind it
#pragma unroll
                for (int t4 = (i + 1) / 4; t4 < kChunkRows / 4; ++t4) {
                    const float4 a = *reinterpret_cast<const float4*>(sa + i * kAStride + 4 * t4);
                    if (4 * t4 > i) x[4 * t4] = fmaf(-a.x, x[i], x[4 * t4]);
                    if (4 * t4 + 1 > i) x[4 * t4 + 1] = fmaf(-a.y, x[i], x[4 * t4 + 1]);
                    if (4 * t4 + 2 > i) x[4 * t4 + 2] = fmaf(-a.z, x[i], x[4 * t4 + 2]);
                    if (4 * t4 + 3 > i) x[4 * t4 + 3] = fmaf(-a.w, x[i], x[4 * t4 + 3]);
                }
            }
            float* to = is_key ? solved_k : values;
            const int width = is_key ? p.dim_p : p.vdim_p;
#pragma unroll
            for (int t = 0; t < kChunkRows; ++t) to[t * width + j] = x[t];
        }
    }
}

// What a wave needs of a chunk, all of it asked for a chunk ahead.
template <bool kDelta, int kT>
struct ChunkOperands {
    float4 w[kDelta ? 4 : 1][kT], q[4][kT], k[kT][4], m[4];
    float u[4], total;
};

template <bool kDelta, int kT>
__device__ inline void fetch_chunk(const ChunkArgs& p, int chunk, int head, int wave, int c, int g, int col, ChunkOperands<kDelta, kT>& o) {
    const long at = static_cast<long>(chunk) * p.heads + head;
    const float* q_in = p.q_in + at * kChunkRows * p.dim_p + 16 * wave * kT + 4 * g;
    const float* k_out = p.k_out + at * kChunkRows * p.dim_p + 4 * g;
#pragma unroll
    for (int t = 0; t < kT; ++t) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            if constexpr (kDelta)
                o.w[r][t] = *reinterpret_cast<const float4*>(p.solved_k + at * kChunkRows * p.dim_p + (16 * r + c) * p.dim_p + 16 * (wave * kT + t) + 4 * g);
            o.q[r][t] = *reinterpret_cast<const float4*>(q_in + (16 * r + c) * p.dim_p + 16 * t);
            o.k[t][r] = *reinterpret_cast<const float4*>(k_out + (16 * (wave * kT + t) + c) * kChunkRows + 16 * r);
        }
    }
#pragma unroll
    for (int s = 0; s < 4; ++s)
        o.m[s] = s <= wave ? *reinterpret_cast<const float4*>(p.mix + at * kChunkRows * kChunkRows + (16 * wave + c) * kChunkRows + 16 * s + 4 * g)
                           : float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int v = 0; v < 4; ++v) o.u[v] = p.values[at * kChunkRows * p.vdim_p + (16 * wave + 4 * g + v) * p.vdim_p + col];
    o.total = p.total[at];
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
        const int first = p.chunks[4 * chunk], n = p.chunks[4 * chunk + 1] - first;
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
            if (t < n && col < p.vdim) p.out[(static_cast<long>(first + t) * p.heads + head) * p.vdim + col] = o[v];
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
    const size_t shared = (2 * kChunkRows * (a.dim_p + 4) + (delta ? kChunkRows * (kChunkRows + 4) : 0)) * sizeof(float);
    static bool allowed = false;
    if (!allowed) {
        const int most = (2 * kChunkRows * (kChunkMaxDim + 4) + kChunkRows * (kChunkRows + 4)) * sizeof(float);
        for (const void* kernel : {reinterpret_cast<const void*>(&chunk_prepare_kernel<false>), reinterpret_cast<const void*>(&chunk_prepare_kernel<true>)}) {
            const hipError_t e = hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, most);
            LEONE_REQUIRE(e == hipSuccess, "chunked_memory: %d bytes of shared memory were refused: %s", most, hipGetErrorString(e));
        }
        allowed = true;
    }
    const dim3 prepare(n_chunks, heads), walk(n_links, heads, a.vdim_p / 16);
    if (delta) {
        chunk_prepare_kernel<true><<<prepare, kChunkThreads, shared, stream>>>(a);
        LEONE_LAUNCH_CHECK("chunk_prepare");
        if (tiles == 1) chunk_walk_kernel<true, 1><<<walk, kChunkThreads, 0, stream>>>(a);
        else chunk_walk_kernel<true, 2><<<walk, kChunkThreads, 0, stream>>>(a);
    } else {
        chunk_prepare_kernel<false><<<prepare, kChunkThreads, shared, stream>>>(a);
        LEONE_LAUNCH_CHECK("chunk_prepare");
        if (tiles == 1) chunk_walk_kernel<false, 1><<<walk, kChunkThreads, 0, stream>>>(a);
        else chunk_walk_kernel<false, 2><<<walk, kChunkThreads, 0, stream>>>(a);
    }
    LEONE_LAUNCH_CHECK("chunk_walk");
    return 0;
}
