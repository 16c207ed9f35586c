// What an attention kernel may do to its scores and results beside the mask, all of it optional.
#pragma once

#include "common.h"

namespace leone {

// The first key that a query at position pos sees: the last `window` positions (0: all), or, with chunks (chunk > 0, then no
// window), the positions of pos's own chunk of so many, counted from position 0.
__device__ inline int first_key(int pos, int window, int chunk) {
    if (chunk > 0) return pos - pos % chunk;
    return (window > 0 && pos - window + 1 > 0) ? pos - window + 1 : 0;
}

// Scores held to a cap (cap > 0: score = cap * tanh(score / cap), taken on the scaled score), a sink in the denominator
// (sinks float [q_heads] or null: exp(sinks[h]) is added once, weighs no value and is neither scaled nor capped), and
// values that were turned by their own position when they were cached: a head's result at position i is turned back by
// i's angles (tables float [turn_positions, v_dim / 2] or null; pairs (m, m + v_dim / 2), or (2 m, 2 m + 1) for
// turn_pairing 1).
struct ScoreShape {
    float cap = 0.f;
    const float* sinks = nullptr;
    const float* turn_cos = nullptr;
    const float* turn_sin = nullptr;
    int turn_positions = 0;
    int turn_pairing = 0;
    bool any() const { return cap > 0.f || sinks != nullptr || turn_cos != nullptr; }
};

// tanh from one power of two and one division: 1 - 2 / (1 + e^(2x)), off by a few 1e-7 of 1.
__device__ inline float tanh_fast(float x) {
    return 1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(x * 2.885390081777926815f));
}

// The pair that element d of a head belongs to, and d's partner in it.
__device__ inline int turn_pair(int d, int half, int pairing) { return pairing ? d >> 1 : (d < half ? d : d - half); }
__device__ inline int turn_partner(int d, int half, int pairing) { return pairing ? d ^ 1 : (d < half ? d + half : d - half); }
__device__ inline bool turn_is_first(int d, int half, int pairing) { return pairing ? (d & 1) == 0 : d < half; }

// Element d of a result turned back at position pos, from its own value and its partner's: (u, v) becomes
// (u cos + v sin, v cos - u sin).
__device__ inline float turned_back(float own, float partner, int d, int v_dim, long pos, const ScoreShape& s) {
    const int half = v_dim / 2, m = turn_pair(d, half, s.turn_pairing);
    const long at = (pos < s.turn_positions ? pos : s.turn_positions - 1) * half + m;
    const float c = s.turn_cos[at], n = s.turn_sin[at];
    return turn_is_first(d, half, s.turn_pairing) ? own * c + partner * n : own * c - partner * n;
}

inline int check_mask(const char* what, int window, int chunk, int keep_first) {
    LEONE_REQUIRE(window >= 0 && chunk >= 0, "%s: window %d and chunk %d must not be negative", what, window, chunk);
    LEONE_REQUIRE(chunk == 0 || (window == 0 && keep_first == 0), "%s: keys are seen by chunks of %d or by a window, not both", what, chunk);
    return 0;
}

inline int check_score_shape(const char* what, const ScoreShape& s, int v_dim) {
    LEONE_REQUIRE(s.cap >= 0.f && s.cap == s.cap, "%s: the scores' cap must not be negative", what);
    LEONE_REQUIRE((s.turn_cos == nullptr) == (s.turn_sin == nullptr), "%s: the tables that turn values back come together", what);
    LEONE_REQUIRE(!s.turn_cos || (s.turn_positions > 0 && v_dim % 2 == 0 && (s.turn_pairing == 0 || s.turn_pairing == 1)),
                  "%s: values of %d elements cannot be turned back by tables of %d positions", what, v_dim, s.turn_positions);
    return 0;
}

}  // namespace leone
