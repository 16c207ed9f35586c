// Attention over the paged cache.
//
// For a query row at absolute position `pos` of its request and query head h,
// with kv head h / (q_heads / kv_heads): scores s_j = (q . K[j]) * scale for
// keys j in [first, pos], first = 0 or pos - window + 1 for a windowed layer, and, if the layer keeps its
// first tokens in sight, also for the keys j < keep_first (at their own places in the cache);
// softmax over them; out = sum_j p_j V[j].  This is the reference's recurrence
// (crates/leone/src/cpu.rs:2299-2421: scale after the dot, running maximum,
// rescaled sum and accumulator), with the keys found through the request's block
// table instead of its segment list.  Scores, maxima, sums and the accumulator
// are float whatever the cache's storage type.
//
// Cache layout of one layer: [page][kv head] blocks of page_tokens * head_dim
// elements, packed inside as key_offset() and value_offset() say.
#include "common.h"
#include "leone_hip.h"
#include "score_shape.h"

#include <math.h>

namespace leone {

constexpr int kRowThreads = 256;
constexpr int kRowWaves = kRowThreads / kWave;
constexpr int kRowDimsPerLane = 4;                      // keys and values of up to 256 elements a head
constexpr int kRowMaxHeadDim = kWave * kRowDimsPerLane;

// One block per (row, query head).  Wave w takes keys first + w, first + w + 4,
// ...; lanes split the head's elements.  The four partial results are merged
// in a fixed order, so a launch repeats bit for bit.
template <typename T>
__global__ void attention_rows_kernel(const T* __restrict__ q, T* __restrict__ out,
                                      const T* __restrict__ k_pool, const T* __restrict__ v_pool,
                                      const int* __restrict__ positions, const int* __restrict__ row_entry,
                                      const int* __restrict__ block_table, int max_blocks, int q_heads,
                                      int kv_heads, int head_dim, int v_dim, int page_tokens, float scale, int window,
                                      const float* __restrict__ gate, long gate_stride, int keep_first, int gate_each,
                                      const float* __restrict__ slopes, float temp_coef, int temp_every, ScoreShape shape, int chunk) {
    __shared__ float sm_m[kRowWaves];
    __shared__ float sm_l[kRowWaves];
    __shared__ float sm_acc[kRowWaves][kRowMaxHeadDim];

    const int row = blockIdx.x;
    const int head = blockIdx.y;
    const int wave = threadIdx.x / kWave;
    const int lane = threadIdx.x % kWave;
    const int kvh = head / (q_heads / kv_heads);
    const int pos = positions[row];
    const int* table = block_table + static_cast<long>(row_entry[row]) * max_blocks;
    const int first = first_key(pos, window, chunk);
    // a query that grows with its position: the factor 1 + coef * ln(floor((pos + 1) / every) + 1) rides on the scale
    if (temp_every > 0) scale *= 1.0f + temp_coef * logf(static_cast<float>((pos + 1) / temp_every + 1));
    // a head's scores are lowered by slope * distance
    const float slope = slopes ? slopes[head] : 0.f;

    const T* qr = q + (static_cast<long>(row) * q_heads + head) * head_dim;
    float qv[kRowDimsPerLane];
#pragma unroll
    for (int i = 0; i < kRowDimsPerLane; ++i) {
        const int d = lane + i * kWave;
        qv[i] = d < head_dim ? to_float(qr[d]) : 0.f;
    }

    float m = -INFINITY, l = 0.f;
    float acc[kRowDimsPerLane];
#pragma unroll
    for (int i = 0; i < kRowDimsPerLane; ++i) acc[i] = 0.f;
    // the kept first keys that the window has left behind come first, then the window's
    const int kept = keep_first < first ? keep_first : first;
    const int reach = kept + pos - first + 1;
    for (int t = wave; t < reach; t += kRowWaves) {
        const int j = t < kept ? t : first + (t - kept);
        const int page = table[j / page_tokens];
        if (page < 0) {  // an unmapped block: poison the result instead of reading outside the pool
            l = __builtin_nanf("");
            continue;
        }
        const T* kr = k_pool + (static_cast<long>(page) * kv_heads + kvh) * page_tokens * head_dim;
        const T* vr = v_pool + (static_cast<long>(page) * kv_heads + kvh) * page_tokens * v_dim;
        const int token = j % page_tokens;
        float partial = 0.f;
        float vv[kRowDimsPerLane];
#pragma unroll
        for (int i = 0; i < kRowDimsPerLane; ++i) {
            const int d = lane + i * kWave;
            if (d < head_dim) partial = fmaf(qv[i], to_float(kr[key_offset(token, d, page_tokens)]), partial);
            vv[i] = d < v_dim ? to_float(vr[value_offset(token, d, v_dim)]) : 0.f;
        }
        float s = wave_sum(partial) * scale;
        if (shape.cap > 0.f) s = shape.cap * tanhf(s / shape.cap);
        s -= slope * static_cast<float>(pos - j);
        const float m_new = fmaxf(m, s);
        const float alpha = expf(m - m_new);
        const float beta = expf(s - m_new);
        l = l * alpha + beta;
#pragma unroll
        for (int i = 0; i < kRowDimsPerLane; ++i) acc[i] = acc[i] * alpha + beta * vv[i];
        m = m_new;
    }
    if (lane == 0) {
        sm_m[wave] = m;
        sm_l[wave] = l;
    }
#pragma unroll
    for (int i = 0; i < kRowDimsPerLane; ++i) sm_acc[wave][lane + i * kWave] = acc[i];
    __syncthreads();

    T* orow = out + (static_cast<long>(row) * q_heads + head) * v_dim;
    // an output gate: the result times sigmoid(gate[row, head]), or, with a gate for each element, times
    // sigmoid(gate[row, head * v_dim + d])
    const float* gate_row = gate ? gate + static_cast<long>(row) * gate_stride + (gate_each ? static_cast<long>(head) * v_dim : head) : nullptr;
    const float open_head = (gate && !gate_each) ? 1.0f / (1.0f + expf(-gate_row[0])) : 1.0f;
    float top = sm_m[0];
#pragma unroll
    for (int w = 1; w < kRowWaves; ++w) top = fmaxf(top, sm_m[w]);
    const float sink = shape.sinks ? shape.sinks[head] : -INFINITY;
    top = fmaxf(top, sink);
    float wgt[kRowWaves], denom = shape.sinks ? expf(sink - top) : 0.f;
#pragma unroll
    for (int w = 0; w < kRowWaves; ++w) {
        // A wave that saw no key has m = -inf and contributes nothing.
        wgt[w] = sm_m[w] == -INFINITY ? 0.f : expf(sm_m[w] - top);
        denom += sm_l[w] * wgt[w];
    }
    auto result = [&](int d) {
        float num = 0.f;
#pragma unroll
        for (int w = 0; w < kRowWaves; ++w) num += sm_acc[w][d] * wgt[w];
        return num / denom;
    };
    for (int d = threadIdx.x; d < v_dim; d += kRowThreads) {
        const float open = (gate && gate_each) ? 1.0f / (1.0f + expf(-gate_row[d])) : open_head;
        float value = result(d);
        if (shape.turn_cos)
            value = turned_back(value, result(turn_partner(d, v_dim / 2, shape.turn_pairing)), d, v_dim, pos, shape);
        orow[d] = from_float<T>(value * open);
    }
}

// The same with the heads' scores mixed before the softmax: score_h <- sum_g talk[h, g] score_g over all query heads g.
// One workgroup per (row, query head h).  A dot product with every kv head's key is one with the queries of that kv head's
// group summed with talk's weights, so the mixed score of head h is one dot product over all kv heads' keys side by side:
// the workgroup makes that query (kv_heads * head_dim floats, in shared memory) and walks the keys as above, the values
// those of h's own kv head.
template <typename T>
__global__ void __launch_bounds__(kRowThreads)
attention_rows_talk_kernel(const T* __restrict__ q, T* __restrict__ out, const T* __restrict__ k_pool, const T* __restrict__ v_pool,
                           AnyVec talk, const int* __restrict__ positions, const int* __restrict__ row_entry,
                           const int* __restrict__ block_table, int max_blocks, int q_heads, int kv_heads, int head_dim,
                           int v_dim, int page_tokens, float scale, int window) {
    __shared__ float sm_m[kRowWaves];
    __shared__ float sm_l[kRowWaves];
    __shared__ float sm_acc[kRowWaves][kRowMaxHeadDim];
    extern __shared__ float mixed_q[];                      // [kv_heads][head_dim]
    const int row = blockIdx.x, head = blockIdx.y;
    const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave;
    const int group = q_heads / kv_heads, kvh = head / group;
    const int pos = positions[row];
    const int* table = block_table + static_cast<long>(row_entry[row]) * max_blocks;
    const int first = (window > 0 && pos - window + 1 > 0) ? pos - window + 1 : 0;
    const T* qr = q + static_cast<long>(row) * q_heads * head_dim;
    for (int e = threadIdx.x; e < kv_heads * head_dim; e += kRowThreads) {
        const int c = e / head_dim, d = e % head_dim;
        float sum = 0.f;
        for (int g = c * group; g < (c + 1) * group; ++g)
            sum = fmaf(load_any(talk, static_cast<long>(head) * q_heads + g), to_float(qr[static_cast<long>(g) * head_dim + d]), sum);
        mixed_q[e] = sum;
    }
    __syncthreads();
    float m = -INFINITY, l = 0.f;
    float acc[kRowDimsPerLane];
#pragma unroll
    for (int i = 0; i < kRowDimsPerLane; ++i) acc[i] = 0.f;
    for (int j = first + wave; j <= pos; j += kRowWaves) {
        const int page = table[j / page_tokens];
        if (page < 0) {  // an unmapped block: poison the result instead of reading outside the pool
            l = __builtin_nanf("");
            continue;
        }
        const T* kr = k_pool + static_cast<long>(page) * kv_heads * page_tokens * head_dim;
        const T* vr = v_pool + (static_cast<long>(page) * kv_heads + kvh) * page_tokens * v_dim;
        const int token = j % page_tokens;
        float partial = 0.f;
        for (int c = 0; c < kv_heads; ++c)
            for (int d = lane; d < head_dim; d += kWave)
                partial = fmaf(mixed_q[c * head_dim + d],
                               to_float(kr[static_cast<long>(c) * page_tokens * head_dim + key_offset(token, d, page_tokens)]), partial);
        float vv[kRowDimsPerLane];
#pragma unroll
        for (int i = 0; i < kRowDimsPerLane; ++i) {
            const int d = lane + i * kWave;
            vv[i] = d < v_dim ? to_float(vr[value_offset(token, d, v_dim)]) : 0.f;
        }
        const float s = wave_sum(partial) * scale;
        const float m_new = fmaxf(m, s);
        const float alpha = expf(m - m_new), beta = expf(s - m_new);
        l = l * alpha + beta;
#pragma unroll
        for (int i = 0; i < kRowDimsPerLane; ++i) acc[i] = acc[i] * alpha + beta * vv[i];
        m = m_new;
    }
    if (lane == 0) {
        sm_m[wave] = m;
        sm_l[wave] = l;
    }
#pragma unroll
    for (int i = 0; i < kRowDimsPerLane; ++i) sm_acc[wave][lane + i * kWave] = acc[i];
    __syncthreads();
    float top = sm_m[0];
#pragma unroll
    for (int w = 1; w < kRowWaves; ++w) top = fmaxf(top, sm_m[w]);
    float wgt[kRowWaves], denom = 0.f;
#pragma unroll
    for (int w = 0; w < kRowWaves; ++w) {
        wgt[w] = sm_m[w] == -INFINITY ? 0.f : expf(sm_m[w] - top);
        denom += sm_l[w] * wgt[w];
    }
    for (int d = threadIdx.x; d < v_dim; d += kRowThreads) {
        float num = 0.f;
#pragma unroll
        for (int w = 0; w < kRowWaves; ++w) num += sm_acc[w][d] * wgt[w];
        out[(static_cast<long>(row) * q_heads + head) * v_dim + d] = from_float<T>(num / denom);
    }
}

}  // namespace leone

using namespace leone;

extern "C" int leone_attention_rows(const void* q, void* out, const void* k_pool, const void* v_pool, int dtype,
                                    const int* positions, const int* row_entry, const int* block_table,
                                    int max_blocks, int rows, int q_heads, int kv_heads, int head_dim, int v_dim,
                                    int page_tokens, float scale, int window, const float* gate, long gate_stride,
                                    hipStream_t stream) {
    return leone_attention_rows_kept(q, out, k_pool, v_pool, dtype, positions, row_entry, block_table, max_blocks, rows,
                                     q_heads, kv_heads, head_dim, v_dim, page_tokens, scale, window, gate, gate_stride, 0, 0, stream);
}

// keep_first: keys at positions below it stay in sight of a windowed layer.  gate_each: the gate holds a value
// for every element of every head ([rows, q_heads * v_dim] within rows of gate_stride) instead of one a head.
extern "C" int leone_attention_rows_kept(const void* q, void* out, const void* k_pool, const void* v_pool, int dtype,
                                         const int* positions, const int* row_entry, const int* block_table,
                                         int max_blocks, int rows, int q_heads, int kv_heads, int head_dim, int v_dim,
                                         int page_tokens, float scale, int window, const float* gate, long gate_stride,
                                         int keep_first, int gate_each, hipStream_t stream) {
    return leone_attention_rows_biased(q, out, k_pool, v_pool, dtype, positions, row_entry, block_table, max_blocks, rows,
                                       q_heads, kv_heads, head_dim, v_dim, page_tokens, scale, window, gate, gate_stride,
                                       keep_first, gate_each, nullptr, 0.f, 0, stream);
}

// slopes (float [q_heads], may be null): head h's score for the key at distance d = pos - j is lowered by slopes[h] * d.
// temp_every > 0: the row's queries count times 1 + temp_coef * ln(floor((pos + 1) / temp_every) + 1).
extern "C" int leone_attention_rows_biased(const void* q, void* out, const void* k_pool, const void* v_pool, int dtype,
                                           const int* positions, const int* row_entry, const int* block_table,
                                           int max_blocks, int rows, int q_heads, int kv_heads, int head_dim, int v_dim,
                                           int page_tokens, float scale, int window, const float* gate, long gate_stride,
                                           int keep_first, int gate_each, const float* slopes, float temp_coef,
                                           int temp_every, hipStream_t stream) {
    return leone_attention_rows_shaped(q, out, k_pool, v_pool, dtype, positions, row_entry, block_table, max_blocks, rows,
                                       q_heads, kv_heads, head_dim, v_dim, page_tokens, scale, window, gate, gate_stride,
                                       keep_first, gate_each, slopes, temp_coef, temp_every, 0.f, nullptr, nullptr, nullptr, 0,
                                       0, 0, stream);
}

// The same with what score_shape.h describes: cap (0: none), sinks, and the tables that turn results back (null: none);
// chunk > 0 (no window, no kept first keys): a row sees the keys of its own chunk of so many positions only.
extern "C" int leone_attention_rows_shaped(const void* q, void* out, const void* k_pool, const void* v_pool, int dtype,
                                           const int* positions, const int* row_entry, const int* block_table,
                                           int max_blocks, int rows, int q_heads, int kv_heads, int head_dim, int v_dim,
                                           int page_tokens, float scale, int window, const float* gate, long gate_stride,
                                           int keep_first, int gate_each, const float* slopes, float temp_coef,
                                           int temp_every, float cap, const float* sinks, const float* turn_cos,
                                           const float* turn_sin, int turn_positions, int turn_pairing, int chunk,
                                           hipStream_t stream) {
    if (check_mask("attention_rows", window, chunk, keep_first)) return 1;
    const ScoreShape shape{cap, sinks, turn_cos, turn_sin, turn_positions, turn_pairing};
    if (check_score_shape("attention_rows", shape, v_dim)) return 1;
    LEONE_REQUIRE(temp_every >= 0, "attention_rows: the query factor's period %d must not be negative", temp_every);
    LEONE_REQUIRE(dtype == kF32 || dtype == kBF16, "attention_rows: unknown element type %d", dtype);
    LEONE_REQUIRE(q && out && k_pool && v_pool && positions && row_entry && block_table, "attention_rows: null pointer");
    LEONE_REQUIRE(rows > 0 && q_heads > 0 && kv_heads > 0 && q_heads % kv_heads == 0,
                  "attention_rows: rows %d, %d query heads over %d kv heads", rows, q_heads, kv_heads);
    LEONE_REQUIRE(q_heads <= 65535, "attention_rows: at most 65535 query heads");
    LEONE_REQUIRE(head_dim > 0 && head_dim <= kRowMaxHeadDim, "attention_rows: head_dim %d must be in 1..%d", head_dim, kRowMaxHeadDim);
    LEONE_REQUIRE(v_dim > 0 && v_dim <= kRowMaxHeadDim, "attention_rows: value size %d must be in 1..%d", v_dim, kRowMaxHeadDim);
    LEONE_REQUIRE(!gate || gate_stride >= (gate_each ? static_cast<long>(q_heads) * v_dim : q_heads),
                  "attention_rows: gate rows of %ld for %d heads", gate_stride, q_heads);
    LEONE_REQUIRE(keep_first >= 0, "attention_rows: keep_first %d must not be negative", keep_first);
    LEONE_REQUIRE(page_tokens > 0 && max_blocks > 0, "attention_rows: page_tokens %d and max_blocks %d must be positive", page_tokens, max_blocks);
    LEONE_REQUIRE(head_dim % 8 == 0 && page_tokens % 8 == 0,
                  "attention_rows: head_dim %d and page_tokens %d must be multiples of 8", head_dim, page_tokens);
    LEONE_REQUIRE(window >= 0, "attention_rows: window %d must not be negative", window);
    dim3 grid(rows, q_heads);
    if (dtype == kF32)
        attention_rows_kernel<float><<<grid, kRowThreads, 0, stream>>>(
            static_cast<const float*>(q), static_cast<float*>(out), static_cast<const float*>(k_pool),
            static_cast<const float*>(v_pool), positions, row_entry, block_table, max_blocks, q_heads, kv_heads,
            head_dim, v_dim, page_tokens, scale, window, gate, gate_stride, keep_first, gate_each, slopes, temp_coef, temp_every, shape, chunk);
    else
        attention_rows_kernel<bf16_t><<<grid, kRowThreads, 0, stream>>>(
            static_cast<const bf16_t*>(q), static_cast<bf16_t*>(out), static_cast<const bf16_t*>(k_pool),
            static_cast<const bf16_t*>(v_pool), positions, row_entry, block_table, max_blocks, q_heads, kv_heads,
            head_dim, v_dim, page_tokens, scale, window, gate, gate_stride, keep_first, gate_each, slopes, temp_coef, temp_every, shape, chunk);
    LEONE_LAUNCH_CHECK("attention_rows");
    return 0;
}

// talk [q_heads, q_heads] of talk_dtype: the heads' scores are mixed by it before the softmax.
extern "C" int leone_attention_rows_talk(const void* q, void* out, const void* k_pool, const void* v_pool, int dtype,
                                         const void* talk, int talk_dtype, const int* positions, const int* row_entry,
                                         const int* block_table, int max_blocks, int rows, int q_heads, int kv_heads,
                                         int head_dim, int v_dim, int page_tokens, float scale, int window, hipStream_t stream) {
    LEONE_REQUIRE((dtype == kF32 || dtype == kBF16) && (talk_dtype == kF32 || talk_dtype == kBF16), "attention_rows_talk: unknown element type");
    LEONE_REQUIRE(q && out && k_pool && v_pool && talk && positions && row_entry && block_table, "attention_rows_talk: null pointer");
    LEONE_REQUIRE(rows > 0 && q_heads > 0 && kv_heads > 0 && q_heads % kv_heads == 0 && q_heads <= 65535,
                  "attention_rows_talk: rows %d, %d query heads over %d kv heads", rows, q_heads, kv_heads);
    LEONE_REQUIRE(head_dim > 0 && head_dim % 8 == 0 && v_dim > 0 && v_dim <= kRowMaxHeadDim,
                  "attention_rows_talk: heads of %d and values of %d elements (at most %d)", head_dim, v_dim, kRowMaxHeadDim);
    LEONE_REQUIRE(page_tokens > 0 && page_tokens % 8 == 0 && max_blocks > 0 && window >= 0, "attention_rows_talk: bad pages or window");
    const size_t shared = static_cast<size_t>(kv_heads) * head_dim * sizeof(float);
    LEONE_REQUIRE(shared <= 56 * 1024, "attention_rows_talk: %d kv heads of %d elements do not fit shared memory", kv_heads, head_dim);
    const dim3 grid(rows, q_heads);
    const AnyVec mix{talk, talk_dtype};
#define LEONE_TALK(T)                                                                                                       \
    attention_rows_talk_kernel<T><<<grid, kRowThreads, shared, stream>>>(                                                   \
        static_cast<const T*>(q), static_cast<T*>(out), static_cast<const T*>(k_pool), static_cast<const T*>(v_pool), mix,  \
        positions, row_entry, block_table, max_blocks, q_heads, kv_heads, head_dim, v_dim, page_tokens, scale, window)
    if (dtype == kF32) LEONE_TALK(float);
    else LEONE_TALK(bf16_t);
#undef LEONE_TALK
    LEONE_LAUNCH_CHECK("attention_rows_talk");
    return 0;
}
