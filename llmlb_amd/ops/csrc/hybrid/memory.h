// What the kernels of matrix memory (mLSTM) share.
#pragma once
#include "common.h"

// floats a head keeps beside its matrix: the normaliser in whole vectors,
// then a vector whose first number is the running maximum
__host__ __device__ __forceinline__ int extra_row(int D) {
  return (D + 3) / 4 * 4 + 4;
}

// Log input and forget gates of one head and token, cap tanh(z / cap) and
// the logarithm of its sigmoid.
__device__ __forceinline__ void memory_gates(float zi, float zf, float cap,
                                             float& li, float& lf) {
  li = cap * tanhf(zi / cap);
  lf = -softplus_f(-cap * tanhf(zf / cap));
}
#define MEMORY_EPS 1e-6f
