// Chunks of 64 rows of the segments of a packed step: what the forms of linear attention over chunks go by.
#pragma once
#include "common.h"

namespace arle {

constexpr int kChunkRows = 64;

struct ChunkAt {
  int seg, row0, rows;   // the request's segment; the chunk's first row in the step; its rows (<= 64), 0: no such chunk
};

// The item-th chunk of all segments, in order.
__device__ __forceinline__ ChunkAt find_chunk(const int* seg_row0, int segments, int item) {
  for (int seg = 0; seg < segments; ++seg) {
    const int a = seg_row0[seg], n = seg_row0[seg + 1] - a, chunks = (n + kChunkRows - 1) / kChunkRows;
    if (item < chunks) return ChunkAt{seg, a + item * kChunkRows, min(kChunkRows, n - item * kChunkRows)};
    item -= chunks;
  }
  return ChunkAt{0, 0, 0};
}

}  // namespace arle
