// Lists of the tokens that each expert serves.
//
// A (token, choice) pair is the number p = token * top + choice.  counts[e]
// is the length of expert e's list, pairs[e * n_tok ..] the list; the order
// of a list does not matter, for every pair's row is computed on its own.
#pragma once
#include "common.h"

// The expert and the tile of BM pairs of its list that workgroup number
// ``tile`` computes, experts one after another; false past the last one.
// Called by whole waves.
struct ExpertTile {
  int expert, first, n;  // n pairs from ``first`` on
};
template <int BM>
__device__ __forceinline__ bool find_tile(const int* counts, int E, int tile,
                                          ExpertTile& out) {
  const int lane = threadIdx.x & (WAVE - 1);
  for (int e0 = 0; e0 < E; e0 += WAVE) {
    const int n = e0 + lane < E ? counts[e0 + lane] : 0;
    const int tiles = (n + BM - 1) / BM;
    int sum = tiles;  // of this lane's and all earlier experts
#pragma unroll
    for (int o = 1; o < WAVE; o *= 2) {
      const int x = __shfl_up(sum, o, WAVE);
      if (lane >= o) sum += x;
    }
    const int all = __shfl(sum, WAVE - 1, WAVE);
    if (tile < all) {
      const unsigned long long past = __ballot(sum > tile);
      const int l = __ffsll((long long)past) - 1;
      const int before = __shfl(sum - tiles, l, WAVE);
      out.expert = e0 + l;
      out.first = (tile - before) * BM;
      out.n = __shfl(n, l, WAVE) - out.first;
      out.n = out.n < BM ? out.n : BM;
      return true;
    }
    tile -= all;
  }
  return false;
}
