// A step's rows cut into chunks: every sequence's new rows in runs of at most `size` rows counted from
// the step's first row of that sequence, sequence after sequence.
#pragma once
#include "common.hpp"

namespace tl {

// chunk c of the step: its sequence, the step's row it starts at and its rows
struct Chunk {
  int b, row0, rows;
};
// false if the step has no chunk c
__device__ __forceinline__ bool find_chunk(int c, const int* cu, int B, int size, Chunk& out) {
  for (int b = 0; b < B; ++b) {
    const int n = cu[b + 1] - cu[b], chunks = (n + size - 1) / size;
    if (c < chunks) {
      out = Chunk{b, cu[b] + c * size, min(size, n - c * size)};
      return true;
    }
    c -= chunks;
  }
  return false;
}

}  // namespace tl
