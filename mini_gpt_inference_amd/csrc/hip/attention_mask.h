// Which keys a query sees, and what is added to its scores by distance: shared by the attention kernels.
#pragma once
#include <hip/hip_runtime.h>

// The first position that a query at position p sees (beside the first positions that a window may keep):
// 0 without a window; with one the last `window` positions; with `chunked` the positions of its own chunk,
// chunks of `window` positions counted from position 0 of the sequence.
__device__ __forceinline__ int first_seen(int p, int window, int chunked) {
  if (window <= 0) return 0;
  if (chunked) return p - p % window;
  return p - window + 1 > 0 ? p - window + 1 : 0;
}

// The number added to the score of a key n positions back: a table of `len` distances (a head's row), whose last
// entry serves every distance beyond.
__device__ __forceinline__ int distance_entry(int n, int len) {
  return n < 0 ? 0 : (n < len ? n : len - 1);
}
