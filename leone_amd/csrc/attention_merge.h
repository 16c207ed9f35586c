// The second kernels of the attentions that cut a row's keys into parts: partial results (float, unnormalised, with the
// reference and the sum of every part) merged in the order of the parts.
#pragma once

#include "common.h"

namespace leone {

// part_acc [rows * q_heads, splits, head_dim], part_ml [rows * q_heads, splits, 2] -> out bfloat16 [rows * q_heads, head_dim].
void launch_attention_reduce(const float* part_acc, const float* part_ml, bf16_t* out, int rows, int q_heads, int head_dim, int splits,
                             hipStream_t stream);
int attention_reduce_max_splits();

// The same for the rows that n_tiles tiles (entry, first row, rows up to 32) name; head_dim up to 256.
void launch_attention_tile_merge(const float* part_acc, const float* part_ml, bf16_t* out, const int* tiles, int n_tiles, int q_heads,
                                 int head_dim, int splits, hipStream_t stream);
int attention_tile_merge_max_splits();

}  // namespace leone
