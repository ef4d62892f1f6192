// What a sublayer leaves for the residual: a float32 tensor [T, W], or parts that are added in ascending order (the
// partial products of a matrix product whose K was split: part p of row t at p * part_stride + t * row_stride), or the
// outputs of the experts that a token chose, [T, n, W] with a weight per (token, part).  `weights` also serves a factor
// per token on all parts (w_part 0).
#pragma once
#include "common.h"

namespace arle {

struct Addend {
  const float* p;         // null: no addend
  int parts;              // parts added in order (>= 1)
  long long part_stride;  // elements between parts of one row
  long long row_stride;   // elements between rows
  const float* weights;   // factor of (row, part) at row * w_row + part * w_part, or null
  int w_row;
  int w_part;
};

}  // namespace arle
