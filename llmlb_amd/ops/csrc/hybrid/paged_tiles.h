// Tiles of keys and values out of the cache's pages, for the matrix-core
// attention kernels of 256 threads.  A page is [G][16 tokens][row].
#pragma once
#include "mfma.h"

// Stages tiles of 64 cached rows of one key/value head, a row being MAPS
// keys of D numbers and a value of V: the keys into lk [64][MAPS DQ + 8],
// the value into lv [64][DV + 8].  A tile starts at a page; a thread's
// pieces of 16 bytes lie in pages that are the same for its whole wave.
template <int MAPS, int DQ, int DV>
struct Stage {
  static constexpr int KP = MAPS * DQ + 8, VP = DV + 8;
  static constexpr int KR = MAPS * DQ / 8, VR = DV / 8;  // pieces of a row
  static constexpr int KL = 64 * KR / 256, VL = 64 * VR / 256;
  static_assert(DQ % 32 == 0 && DV % 32 == 0, "whole waves a page");
  const bf16_t* cache;
  const int* pages;
  size_t page_size;
  int width, D, V, head_off, last_key, last_page;

  __device__ __forceinline__ Stage(const bf16_t* cache_, const int* pages_,
                                   int G, int g, int D_, int V_,
                                   int last_key_)
      : cache(cache_), pages(pages_), width(MAPS * D_ + V_), D(D_), V(V_),
        last_key(last_key_), last_page(last_key_ / PAGE) {
    page_size = (size_t)G * PAGE * width;
    head_off = g * PAGE * width;
  }
  // page numbers of the 64 keys from j0 on
  __device__ __forceinline__ void fetch_pages(int j0,
                                              int (&pg)[4]) const {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int p = j0 / PAGE + i;
      pg[i] = pages[p < last_page ? p : last_page];
    }
  }
  // row r of the fetched tile; r / 16 is the same for the whole wave
  __device__ __forceinline__ const bf16_t* row(int r,
                                               const int (&pg)[4]) const {
    const int s = __builtin_amdgcn_readfirstlane(r / PAGE);
    const int p = s == 0 ? pg[0] : (s == 1 ? pg[1] : (s == 2 ? pg[2]
                                                             : pg[3]));
    return cache + (size_t)__builtin_amdgcn_readfirstlane(p) * page_size +
           head_off + (r % PAGE) * width;
  }
  __device__ __forceinline__ void fetch(int j0, const int (&pg)[4],
                                        u32x4 (&pk)[KL],
                                        u32x4 (&pv)[VL]) const {
#pragma unroll
    for (int i = 0; i < KL; ++i) {
      const int p = threadIdx.x + i * 256;
      const int c = p % KR, d = c % (DQ / 8) * 8;
      // columns past D meet zeros of the query
      pk[i] = *reinterpret_cast<const u32x4*>(
          row(p / KR, pg) + c / (DQ / 8) * D + (d < D ? d : 0));
    }
#pragma unroll
    for (int i = 0; i < VL; ++i) {
      const int p = threadIdx.x + i * 256;
      const int r = p / VR, d = p % VR * 8;
      pv[i] = *reinterpret_cast<const u32x4*>(row(r, pg) + MAPS * D +
                                              (d < V ? d : 0));
      // columns past V are zeros; rows past the last key meet zero weights
      // and must be finite
      if (j0 + r > last_key || d >= V) pv[i] = u32x4{0, 0, 0, 0};
    }
  }
  static __device__ __forceinline__ void store(unsigned short* lk,
                                               unsigned short* lv,
                                               const u32x4 (&pk)[KL],
                                               const u32x4 (&pv)[VL]) {
#pragma unroll
    for (int i = 0; i < KL; ++i) {
      const int p = threadIdx.x + i * 256;
      *reinterpret_cast<u32x4*>(&lk[p / KR * KP + p % KR * 8]) = pk[i];
    }
#pragma unroll
    for (int i = 0; i < VL; ++i) {
      const int p = threadIdx.x + i * 256;
      *reinterpret_cast<u32x4*>(&lv[p / VR * VP + p % VR * 8]) = pv[i];
    }
  }
};
