// Products of tokens with their experts' matrices, any sizes and either
// type: for every pair of an expert's list (experts.h)
//   out[pair] = act(w[expert] in[pair / div])
// with act(z) = max(z, 0)^2 or none.  Tiles of 32 pairs x 64 outputs.
#include "experts.h"

#define BM 32
#define BN 64
#define BK 32

template <typename T>
__global__ __launch_bounds__(256) void expert_rows_kernel(
    T* __restrict__ out, const T* __restrict__ in, const T* __restrict__ w,
    const int* __restrict__ counts, const int* __restrict__ pairs, int E,
    int N, int K, int div, int act, int n_tok) {
  __shared__ float la[BM][BK + 1], lb[BN][BK + 1];
  __shared__ ExpertTiles<BM> tiles;
  if (threadIdx.x < WAVE) tiles.count(counts, E);
  __syncthreads();
  const int i = blockIdx.x, whole = tiles.whole[E - 1];
  if (i >= whole + tiles.rest[E - 1]) return;
  const ExpertTile t =
      tiles.get(counts, E, i < whole ? i : i - whole, i >= whole);
  const int* list = pairs + (size_t)t.expert * n_tok + t.first;
  const T* we = w + (size_t)t.expert * N * K;
  const int n0 = blockIdx.y * BN;
  const int tid = threadIdx.x, r = tid / 8, c = tid % 8;
  const int kr = tid % BK, rr = tid / BK;  // staging: column, first row
  float acc[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) acc[i] = 0.f;
  for (int k0 = 0; k0 < K; k0 += BK) {
    const bool in_k = k0 + kr < K;
#pragma unroll
    for (int i = 0; i < BM; i += 256 / BK)
      la[rr + i][kr] =
          in_k && rr + i < t.n
              ? to_f(in[(size_t)(list[rr + i] / div) * K + k0 + kr])
              : 0.f;
#pragma unroll
    for (int i = 0; i < BN; i += 256 / BK)
      lb[rr + i][kr] = in_k && n0 + rr + i < N
                           ? to_f(we[(size_t)(n0 + rr + i) * K + k0 + kr])
                           : 0.f;
    __syncthreads();
    for (int k = 0; k < BK; ++k) {
      const float a = la[r][k];
#pragma unroll
      for (int i = 0; i < 8; ++i) acc[i] += a * lb[c + i * 8][k];
    }
    __syncthreads();
  }
  if (r >= t.n) return;
  T* dst = out + (size_t)list[r] * N + n0;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    float x = acc[i];
    if (act) {
      x = fmaxf(x, 0.f);
      x *= x;
    }
    if (n0 + c + i * 8 < N) dst[c + i * 8] = from_f<T>(x);
  }
}

extern "C" int hy_expert_rows(void* out, const void* in, const void* w,
                              const void* counts, const void* pairs, int E,
                              int N, int K, int div, int act, int n_tok,
                              int n_pairs, int dtype, void* stream) {
  if (E <= 0 || E > EXPERTS_MAX || N <= 0 || K <= 0 || div <= 0 || N > 65535 * BN) return -2;
  if (n_tok <= 0 || n_pairs <= 0) return 0;
  const int tiles = n_pairs / BM + (E < n_pairs ? E : n_pairs);
  HY_DTYPE(dtype, hipLaunchKernelGGL(
      expert_rows_kernel<T>, dim3(tiles, (N + BN - 1) / BN), dim3(256), 0,
      (hipStream_t)stream, (T*)out, (const T*)in, (const T*)w,
      (const int*)counts, (const int*)pairs, E, N, K, div, act, n_tok));
  HY_CHECK();
  return 0;
}
