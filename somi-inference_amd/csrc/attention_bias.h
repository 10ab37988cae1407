// A learned bias by distance on attention scores: head h adds table[h, n] to the scaled score of the key n positions
// back.  A softmax does not see what is added to all of its scores, so the table is kept relative to its value for far
// keys: it covers the distances 0 .. length - 1 with a last entry of 0, and that entry stands for every key farther
// back.  A kernel then has work with the bias only where a query meets its nearest keys.
#pragma once
#include <hip/hip_runtime.h>

struct DistanceBias {
    const float* table;      // [heads, length] float32 in the units of the scaled scores
    int length;              // 0: no bias
    int in_lds;              // the kernel keeps its heads' rows in LDS (they fit), else it reads the table itself
};

#define BIAS_LDS_FLOATS (10 * 1024)      // floats of the table that a workgroup keeps in LDS at most

// The entry of a key n positions back (a key ahead of the query, which is masked anyway, gets some entry).
__device__ __forceinline__ int bias_index(int n, int length) { return min(max(n, 0), length - 1); }
