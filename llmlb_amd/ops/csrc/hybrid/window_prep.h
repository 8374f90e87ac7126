// Queries and keys of windowed attention before they meet: normed over the
// whole projection, rotated, the keys and values put into the pages.
#pragma once
#include "common.h"

struct WindowPrep {
  void* proj;   // [n_tok][ld]: queries first, keys and values at offsets
  void* cache;
  const float* wq;  // [H D], [G D]
  const float* wk;
  const float* cos_sin;  // [positions][rot], cosines first
  const int* pos;
  const int* row;
  const int* bt;
  int ld, k_off, v_off, H, G, D, V, rot, max_blocks, n_tok;
  float eps;
};

__host__ inline bool window_prep_ok(const WindowPrep& a) {
  return a.H > 0 && a.G > 0 && a.D > 0 && a.V > 0 && a.rot >= 0 &&
         a.rot <= a.D && a.rot % 2 == 0 && (a.rot == 0 || a.cos_sin) &&
         a.H * a.D <= 16384 && a.G * a.D <= 16384;
}

// One section (queries or keys) of a token in a wave, as units of two
// pieces of 8: a piece and the one it is rotated with, or two neighbours
// past the rotated part.  A lane keeps K units.
template <int K>
struct PrepUnits {
  float lo[K][8], hi[K][8];

  // numbers of unit u: first piece at ``at``, the other ``step`` further
  static __device__ __forceinline__ void place(int u, int D, int rot, int& at,
                                               int& step, int& d) {
    const int per = D / 16, head = u / per, i = u % per;
    const bool turned = i < rot / 16;
    d = turned ? i * 8 : rot + (i - rot / 16) * 16;
    step = turned ? rot / 2 : 8;
    at = head * D + d;
  }
  template <typename T>
  __device__ __forceinline__ float load(const T* src, int units, int lane,
                                        int D, int rot) {
    float ssq = 0.f;
#pragma unroll
    for (int n = 0; n < K; ++n) {
      const int u = lane + n * WAVE;
      if (u < units) {
        int at, step, d;
        place(u, D, rot, at, step, d);
        load8(src + at, lo[n]);
        load8(src + at + step, hi[n]);
#pragma unroll
        for (int j = 0; j < 8; ++j)
          ssq += lo[n][j] * lo[n][j] + hi[n][j] * hi[n][j];
      }
    }
    return ssq;
  }
  // store(number of the piece's first element, piece)
  template <typename F>
  __device__ __forceinline__ void finish(const float* w, float r,
                                         const float* cs, int units, int lane,
                                         int D, int rot, F store) {
#pragma unroll
    for (int n = 0; n < K; ++n) {
      const int u = lane + n * WAVE;
      if (u < units) {
        int at, step, d;
        place(u, D, rot, at, step, d);
        float a[8], b[8];
        load8(w + at, a);
        load8(w + at + step, b);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          a[j] *= lo[n][j] * r;
          b[j] *= hi[n][j] * r;
        }
        if (d < rot) {
          float c[8], s[8];
          load8(cs + d, c);
          load8(cs + rot / 2 + d, s);
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            const float x = a[j];
            a[j] = x * c[j] - b[j] * s[j];
            b[j] = b[j] * c[j] + x * s[j];
          }
        }
        store(at, a);
        store(at + step, b);
      }
    }
  }
};

// One wave a token; KQ and KK units of queries and keys a lane.
template <typename T, int KQ, int KK>
__device__ __forceinline__ void window_prep_wave(const WindowPrep& a, int t) {
  const int lane = threadIdx.x & (WAVE - 1);
  const int pos = a.pos[t], G = a.G, D = a.D, V = a.V;
  T* src = (T*)a.proj + (size_t)t * a.ld;
  const int page = a.bt[(size_t)a.row[t] * a.max_blocks + pos / PAGE];
  T* rows = (T*)a.cache + ((size_t)page * G * PAGE + pos % PAGE) * (D + V);
  const size_t head_step = (size_t)PAGE * (D + V);
  const int uq = a.H * D / 16, uk = G * D / 16;
  PrepUnits<KQ> q;
  PrepUnits<KK> k;
  const float sq = wave_sum(q.load(src, uq, lane, D, a.rot));
  const float sk = wave_sum(k.load(src + a.k_off, uk, lane, D, a.rot));
  for (int i = lane; i < G * (V / 8); i += WAVE) {
    const int g = i / (V / 8), d = i % (V / 8) * 8;
    float f[8];
    load8(src + a.v_off + i * 8, f);
    store8(rows + g * head_step + D + d, f);
  }
  const float* cs = a.cos_sin + (size_t)pos * a.rot;
  k.finish(a.wk, 1.f / sqrtf(sk / (G * D) + a.eps), cs, uk, lane, D, a.rot,
           [&](int at, const float* f) {
             store8(rows + at / D * head_step + at % D, f);
           });
  q.finish(a.wq, 1.f / sqrtf(sq / (a.H * D) + a.eps), cs, uq, lane, D, a.rot,
           [&](int at, const float* f) { store8(src + at, f); });
}

// sizes that window_prep_wave takes with some KQ <= 8, KK <= KQ
__host__ inline bool window_prep_wave_ok(const WindowPrep& a) {
  return a.D % 16 == 0 && a.V % 8 == 0 && a.rot % 16 == 0 && a.ld % 8 == 0 &&
         a.k_off % 8 == 0 && a.v_off % 8 == 0 && a.H * a.D <= 8192 &&
         a.G <= a.H;
}

// GO(KQ, KK) for q and k numbers of a token's queries and keys
#define WINDOW_PREP_UNITS(q, k)                                              \
  do {                                                                       \
    const bool few = (k) <= 1024;                                            \
    if ((q) <= 1024) GO(1, 1);                                               \
    else if ((q) <= 2048) { if (few) GO(2, 1); else GO(2, 2); }              \
    else if ((q) <= 4096) { if (few) GO(4, 1); else GO(4, 4); }              \
    else { if (few) GO(8, 1); else GO(8, 8); }                               \
  } while (0)
