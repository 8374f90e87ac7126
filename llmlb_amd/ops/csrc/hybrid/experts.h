// Lists of the tokens that each expert serves.
//
// A (token, choice) pair is the number p = token * top + choice.  counts[e]
// is the length of expert e's list, pairs[e * n_tok ..] the list; the order
// of a list does not matter, for every pair's row is computed on its own.
#pragma once
#include "common.h"

// A tile is BM pairs of one expert's list, or what remains of it.  All whole
// tiles are numbered first, expert after expert, then the remainders: they
// are the quick ones, and come last.
struct ExpertTile {
  int expert, first, n;  // n pairs from ``first`` on
};
#define EXPERTS_MAX 1024

template <int BM>
struct ExpertTiles {
  // tiles of the experts up to and with each: whole ones, remainders
  int whole[EXPERTS_MAX], rest[EXPERTS_MAX];

  // one wave
  __device__ __forceinline__ void count(const int* counts, int E) {
    const int lane = threadIdx.x & (WAVE - 1);
    int w0 = 0, r0 = 0;
    for (int e0 = 0; e0 < E; e0 += WAVE) {
      const int n = e0 + lane < E ? counts[e0 + lane] : 0;
      int w = n / BM, r = n % BM != 0;
#pragma unroll
      for (int o = 1; o < WAVE; o *= 2) {
        const int x = __shfl_up(w, o, WAVE), y = __shfl_up(r, o, WAVE);
        if (lane >= o) {
          w += x;
          r += y;
        }
      }
      if (e0 + lane < E) {
        whole[e0 + lane] = w0 + w;
        rest[e0 + lane] = r0 + r;
      }
      w0 += __shfl(w, WAVE - 1, WAVE);
      r0 += __shfl(r, WAVE - 1, WAVE);
    }
  }
  // first expert with ends[e] > i, by whole waves
  static __device__ __forceinline__ int find(const int* ends, int E, int i) {
    const int lane = threadIdx.x & (WAVE - 1);
    for (int e0 = 0; e0 < E; e0 += WAVE) {
      const unsigned long long past =
          __ballot(e0 + lane < E && ends[e0 + lane] > i);
      if (past)
        return __builtin_amdgcn_readfirstlane(
            e0 + __ffsll((long long)past) - 1);
    }
    return E - 1;
  }
  // whole waves: tile i of the whole ones, or of the remainders
  __device__ __forceinline__ ExpertTile get(const int* counts, int E, int i,
                                            bool is_rest) const {
    ExpertTile t;
    t.expert = find(is_rest ? rest : whole, E, i);
    const int before = t.expert ? whole[t.expert - 1] : 0;
    t.first = (is_rest ? whole[t.expert] - before : i - before) * BM;
    t.n = is_rest ? counts[t.expert] - t.first : BM;
    return t;
  }
};
