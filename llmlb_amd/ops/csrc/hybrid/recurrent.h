// Pieces shared by the recurrent layers: short convolutions over packed
// tokens, runs of neighbouring elements, rows of a state.
//
// A state is [slots][H][V][D] float, value-major: 16 neighbouring lanes
// hold one value column, rows_per_lane(D) key channels each, and read it
// in one run.  A convolution's last inputs are a ring [slots][taps][C],
// position p in entry p % taps: the entry of the current token is never
// one that its own taps read.
#pragma once
#include "common.h"

// silu(conv + bias) of channel c at packed token t (bias null: none)
template <typename T>
__device__ __forceinline__ float conv_silu(
    const T* __restrict__ proj, int ld, const T* __restrict__ ring,
    const float* __restrict__ wconv, const float* __restrict__ bias, int C,
    int taps, int c, int t, int pos, int tstart, int slot) {
  float acc = to_f(proj[(size_t)t * ld + c]) *
                  wconv[(size_t)(taps - 1) * C + c] +
              (bias ? bias[c] : 0.f);
  for (int back = 1; back < taps; ++back) {
    const int p = pos - back;
    if (p < 0) break;
    const float in =
        t - back >= tstart
            ? to_f(proj[(size_t)(t - back) * ld + c])
            : to_f(ring[((size_t)slot * taps + p % taps) * C + c]);
    acc += in * wconv[(size_t)(taps - 1 - back) * C + c];
  }
  return silu_f(acc);
}

// N consecutive elements, as wide as alignment allows; VEC: the address
// is aligned to the whole run (or to 16 bytes).
template <int N, bool VEC>
__device__ __forceinline__ void load_run(const bf16_t* p, float* f) {
  if (VEC && N % 8 == 0) {
#pragma unroll
    for (int i = 0; i < N; i += 8) load8(p + i, f + i);
  } else if (VEC && N == 4) {
    load4(p, f);
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) f[i] = to_f(p[i]);
  }
}
template <int N, bool VEC>
__device__ __forceinline__ void load_run(const float* p, float* f) {
  if (VEC && N % 4 == 0) {
#pragma unroll
    for (int i = 0; i < N; i += 4) load4(p + i, f + i);
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) f[i] = p[i];
  }
}
template <int N, bool VEC>
__device__ __forceinline__ void store_run(float* p, const float* f) {
  if (VEC && N % 4 == 0) {
#pragma unroll
    for (int i = 0; i < N; i += 4) store4(p + i, f + i);
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) p[i] = f[i];
  }
}
template <int N, bool VEC>
__device__ __forceinline__ void store_run(bf16_t* p, const float* f) {
  if (VEC && N % 8 == 0) {
#pragma unroll
    for (int i = 0; i < N; i += 8) store8(p + i, f + i);
  } else if (VEC && N == 4) {
    store4(p, f);
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) p[i] = from_f<bf16_t>(f[i]);
  }
}
// only the first ``valid`` of N elements exist
template <int N, bool VEC, typename T>
__device__ __forceinline__ void load_some(const T* p, int valid, float* f) {
  if (VEC || valid >= N) {
    load_run<N, VEC>(p, f);
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) f[i] = i < valid ? to_f(p[i]) : 0.f;
  }
}
template <int N, bool VEC, typename T>
__device__ __forceinline__ void store_some(T* p, int valid, const float* f) {
  if (VEC || valid >= N) {
    store_run<N, VEC>(p, f);
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i)
      if (i < valid) p[i] = from_f<T>(f[i]);
  }
}

// 16-bit results take the hardware's exponential and logarithm
template <typename T>
__device__ __forceinline__ float sigmoid_t(float x) {
  return sizeof(T) == 2 ? 1.f / (1.f + __expf(-x)) : sigmoid_f(x);
}
template <typename T>
__device__ __forceinline__ float decay_t(float z, float rate) {
  if (sizeof(T) == 2) {
    const float e = __expf(-fabsf(z));
    // log(1 + e) by its series where 1 + e would lose e
    const float lp = e < 1e-3f ? e * (1.f - 0.5f * e) : __logf(1.f + e);
    return __expf(-rate * (fmaxf(z, 0.f) + lp));
  }
  return expf(-rate * softplus_f(z));
}

// The convolution of N neighbouring channels over consecutive tokens,
// each input read once: ``hist`` holds the last taps - 1 inputs.
#define TAPS_MAX 4
template <typename T, int N, bool VEC>
struct ConvRun {
  float w[TAPS_MAX][N], hist[TAPS_MAX - 1][N], b0[N];
  const T* proj;
  const T* ring;
  int ld, C, taps, c, valid;

  __device__ __forceinline__ ConvRun(const T* proj_, int ld_, const T* ring_,
                                     const float* wconv, const float* bias,
                                     int C_, int taps_, int c_, int valid_)
      : proj(proj_), ring(ring_), ld(ld_), C(C_), taps(taps_), c(c_),
        valid(valid_) {
#pragma unroll
    for (int b = 0; b < TAPS_MAX; ++b)
      if (b < taps)
        load_some<N, VEC>(wconv + (size_t)(taps - 1 - b) * C + c, valid,
                          w[b]);
#pragma unroll
    for (int i = 0; i < N; ++i) b0[i] = 0.f;
    if (bias) load_some<N, VEC>(bias + c, valid, b0);
  }
  // inputs before token t, from the batch or the sequence's ring
  __device__ __forceinline__ void start(int t, int pos, int tstart,
                                        int slot) {
#pragma unroll
    for (int b = 1; b < TAPS_MAX; ++b) {
#pragma unroll
      for (int i = 0; i < N; ++i) hist[b - 1][i] = 0.f;
      if (b < taps && pos - b >= 0)
        load_some<N, VEC>(
            t - b >= tstart
                ? proj + (size_t)(t - b) * ld + c
                : ring + ((size_t)slot * taps + (pos - b) % taps) * C + c,
            valid, hist[b - 1]);
    }
  }
  __device__ __forceinline__ void step(int t, float* y) {
    float x[N];
    load_some<N, VEC>(proj + (size_t)t * ld + c, valid, x);
#pragma unroll
    for (int i = 0; i < N; ++i) {
      float acc = x[i] * w[0][i] + b0[i];
#pragma unroll
      for (int b = 1; b < TAPS_MAX; ++b)
        if (b < taps) acc += hist[b - 1][i] * w[b][i];
#pragma unroll
      for (int b = TAPS_MAX - 1; b > 1; --b) hist[b - 1][i] = hist[b - 2][i];
      hist[0][i] = x[i];
      y[i] = acc * sigmoid_t<T>(acc);
    }
  }
};

template <int RPL, bool EXACT>
__device__ __forceinline__ void load_rows(const float* __restrict__ p, int r0,
                                          int D, float* f) {
  if (EXACT && RPL % 4 == 0) {
#pragma unroll
    for (int i = 0; i < RPL / 4; ++i) {
      const float4 v = reinterpret_cast<const float4*>(p + r0)[i];
      f[i * 4] = v.x; f[i * 4 + 1] = v.y;
      f[i * 4 + 2] = v.z; f[i * 4 + 3] = v.w;
    }
  } else {
#pragma unroll
    for (int i = 0; i < RPL; ++i)
      f[i] = (EXACT || r0 + i < D) ? p[r0 + i] : 0.f;
  }
}

template <int RPL, bool EXACT>
__device__ __forceinline__ void store_rows(float* __restrict__ p, int r0,
                                           int D, const float* f) {
  if (EXACT && RPL % 4 == 0) {
#pragma unroll
    for (int i = 0; i < RPL / 4; ++i)
      reinterpret_cast<float4*>(p + r0)[i] =
          make_float4(f[i * 4], f[i * 4 + 1], f[i * 4 + 2], f[i * 4 + 3]);
  } else {
#pragma unroll
    for (int i = 0; i < RPL; ++i)
      if (EXACT || r0 + i < D) p[r0 + i] = f[i];
  }
}

// key channels a lane holds when 16 lanes share a column of D
static int rows_per_lane(int D) {
  int r = 1;
  while (r * 16 < D) r *= 2;
  return r;
}

#define HY_RPL(D, ...)                                                  \
  do {                                                                  \
    const int rpl__ = rows_per_lane(D);                                 \
    const bool ex__ = rpl__ * 16 == (D);                                \
    if (rpl__ == 1) { constexpr int RPL = 1; HY_EX(__VA_ARGS__); }      \
    else if (rpl__ == 2) { constexpr int RPL = 2; HY_EX(__VA_ARGS__); } \
    else if (rpl__ == 4) { constexpr int RPL = 4; HY_EX(__VA_ARGS__); } \
    else if (rpl__ == 8) { constexpr int RPL = 8; HY_EX(__VA_ARGS__); } \
    else if (rpl__ == 16) { constexpr int RPL = 16; HY_EX(__VA_ARGS__); } \
    else { constexpr int RPL = 32; HY_EX(__VA_ARGS__); }                \
  } while (0)
#define HY_EX(...)                                        \
  if (ex__) { constexpr bool EXACT = true; __VA_ARGS__; } \
  else { constexpr bool EXACT = false; __VA_ARGS__; }
