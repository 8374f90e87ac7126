// Differential attention over pages: two score maps per head over the
// same values, out = gate * gain * norm(a1 - lam a2), all in one pass.
//
// A cached token keeps, for each of G key/value heads, one row
//   [key of map 1 (D) | key of map 2 (D) | value (V)];
// a page is [G][16 tokens][2 D + V].  Query head h reads key/value head
// h / (H / G).  q_scale[p] is the score factor of a query at position p;
// scores are bounded to cap tanh(score / cap) where cap > 0.
#include "common.h"

// Copy the keys and values of packed tokens into their pages.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void pair_append_kernel(
    T* __restrict__ cache, const T* __restrict__ proj, int ld, int k_off,
    int v_off, int G, int D, int V, const int* __restrict__ pos_,
    const int* __restrict__ row_, const int* __restrict__ bt, int max_blocks,
    int n_tok) {
  constexpr int N = VEC ? 8 : 1;
  const int width = 2 * D + V;
  const int pieces = width / N, per_tok = G * pieces;
  const long long total = (long long)n_tok * per_tok;
  const long long step = (long long)gridDim.x * 256;
  for (long long id = (long long)blockIdx.x * 256 + threadIdx.x; id < total;
       id += step) {
    const int t = (int)(id / per_tok);
    const int i = (int)(id - (long long)t * per_tok);
    const int g = i / pieces, d = (i - g * pieces) * N;
    const int pos = pos_[t];
    const int page = bt[(size_t)row_[t] * max_blocks + pos / PAGE];
    const T* src = proj + (size_t)t * ld +
                   (d < 2 * D ? k_off + g * 2 * D + d
                              : v_off + g * V + (d - 2 * D));
    T* dst = cache + (((size_t)page * G + g) * PAGE + pos % PAGE) * width + d;
    if (VEC) {
      float f[8];
      load8(src, f);
      store8(dst, f);
    } else {
      dst[0] = src[0];
    }
  }
}

// cap tanh(s / cap); no cap: s
__device__ __forceinline__ float capped(float s, float cap) {
  return cap > 0.f ? cap * tanhf(s / cap) : s;
}

// Any sizes, 32-bit arithmetic: one workgroup per (query, head).  256 keys
// at a time, a thread scores one of them for both maps; then CW threads
// take the value columns of every (256 / CW)th key each.
template <typename T, int NC>
__global__ __launch_bounds__(256) void pair_rows_kernel(
    T* __restrict__ out, int ld_out, const T* __restrict__ proj, int ld,
    int g_off, const T* __restrict__ cache, const int* __restrict__ pos_,
    const int* __restrict__ row_, const int* __restrict__ bt, int max_blocks,
    int H, int G, int D, int V, int CW, const float* __restrict__ q_scale,
    float cap, float lam, float gain, float eps, bool vec) {
  extern __shared__ float lds[];
  float* lq = lds;              // 2 D query numbers
  float* lp = lq + 2 * D;       // weights, 2 x 256
  int* lrow = (int*)(lp + 512); // rows of the keys
  float* lacc = (float*)(lrow + 256);  // 256 x NC x 2
  __shared__ float red[2][4], red2[2][4], red3[4];
  const int t = blockIdx.x, h = blockIdx.y, g = h / (H / G);
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & (WAVE - 1);
  const int pos = pos_[t];
  const int* pages = bt + (size_t)row_[t] * max_blocks;
  const int width = 2 * D + V;
  const T* q = proj + (size_t)t * ld + (size_t)h * 2 * D;
  for (int i = tid; i < 2 * D; i += 256) lq[i] = to_f(q[i]);
  const float scale = q_scale[pos];
  const int grp = tid / CW, ngrp = 256 / CW, c0 = tid % CW;
  float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};
  float acc[2][NC];
#pragma unroll
  for (int i = 0; i < NC; ++i) acc[0][i] = acc[1][i] = 0.f;
  __syncthreads();
  for (int j0 = 0; j0 <= pos; j0 += 256) {
    const int j = j0 + tid;
    float s[2] = {-INFINITY, -INFINITY};
    if (j <= pos) {
      const int row = (pages[j / PAGE] * G + g) * PAGE + j % PAGE;
      lrow[tid] = row;
      const T* k = cache + (size_t)row * width;
      float a = 0.f, b = 0.f;
      if (vec) {
        for (int d = 0; d < D; d += 4) {
          float f[4];
          load4(k + d, f);
#pragma unroll
          for (int i = 0; i < 4; ++i) a += f[i] * lq[d + i];
          load4(k + D + d, f);
#pragma unroll
          for (int i = 0; i < 4; ++i) b += f[i] * lq[D + d + i];
        }
      } else {
        for (int d = 0; d < D; ++d) {
          a += to_f(k[d]) * lq[d];
          b += to_f(k[D + d]) * lq[D + d];
        }
      }
      s[0] = capped(a * scale, cap);
      s[1] = capped(b * scale, cap);
    }
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      float x = s[n];
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) x = fmaxf(x, __shfl_xor(x, o, WAVE));
      if (lane == 0) red[n][wave] = x;
    }
    __syncthreads();
    float keep[2];
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      const float x = fmaxf(fmaxf(fmaxf(red[n][0], red[n][1]),
                                  fmaxf(red[n][2], red[n][3])), m[n]);
      keep[n] = expf(m[n] - x);
      m[n] = x;
      const float p = expf(s[n] - x);
      l[n] = l[n] * keep[n] + p;
      lp[n * 256 + tid] = p;
    }
    __syncthreads();
    const int n_keys = pos - j0 + 1 < 256 ? pos - j0 + 1 : 256;
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      acc[0][i] *= keep[0];
      acc[1][i] *= keep[1];
    }
    for (int k = grp; k < n_keys; k += ngrp) {
      const T* v = cache + (size_t)lrow[k] * width + 2 * D;
#pragma unroll
      for (int i = 0; i < NC; ++i) {
        const int c = c0 + i * CW;
        const float x = c < V ? to_f(v[c]) : 0.f;
        acc[0][i] += lp[k] * x;
        acc[1][i] += lp[256 + k] * x;
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int n = 0; n < 2; ++n) {
    l[n] = wave_sum(l[n]);
    if (lane == 0) red2[n][wave] = l[n];
#pragma unroll
    for (int i = 0; i < NC; ++i) lacc[(n * NC + i) * 256 + tid] = acc[n][i];
  }
  __syncthreads();
  const float i1 =
      1.f / (red2[0][0] + red2[0][1] + red2[0][2] + red2[0][3]);
  const float i2 =
      lam / (red2[1][0] + red2[1][1] + red2[1][2] + red2[1][3]);
  float o[NC], ssq = 0.f;
  if (grp == 0) {
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      float a = 0.f, b = 0.f;
      for (int k = 0; k < ngrp; ++k) {
        a += lacc[i * 256 + k * CW + c0];
        b += lacc[(NC + i) * 256 + k * CW + c0];
      }
      o[i] = c0 + i * CW < V ? a * i1 - b * i2 : 0.f;
      ssq += o[i] * o[i];
    }
  }
  const float r = gain / sqrtf(block_sum_256(ssq, red3) / V + eps);
  if (grp != 0) return;
  const T* gate = proj + (size_t)t * ld + g_off + (size_t)h * V;
  T* dst = out + (size_t)t * ld_out + (size_t)h * V;
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = c0 + i * CW;
    if (c < V) dst[c] = from_f<T>(o[i] * r * sigmoid_f(to_f(gate[c])));
  }
}

extern "C" {

int hy_pair_append(void* cache, const void* proj, int ld, int k_off,
                   int v_off, int G, int D, int V, const void* pos,
                   const void* row, const void* bt, int max_blocks,
                   int n_tok, int dtype, void* stream) {
  if (G <= 0 || D <= 0 || V <= 0) return -2;
  if (n_tok <= 0) return 0;
  const bool vec = D % 8 == 0 && V % 8 == 0 && ld % 8 == 0 &&
                   k_off % 8 == 0 && v_off % 8 == 0;
  const long long work = (long long)n_tok * G * (2 * D + V) / (vec ? 8 : 1);
  const long long blocks = (work + 255) / 256;
  const int grid = (int)(blocks < 8192 ? (blocks > 0 ? blocks : 1) : 8192);
#define GO(VEC)                                                              \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                        \
      (pair_append_kernel<T, VEC>), dim3(grid), dim3(256), 0,                \
      (hipStream_t)stream, (T*)cache, (const T*)proj, ld, k_off, v_off, G, D, \
      V, (const int*)pos, (const int*)row, (const int*)bt, max_blocks,       \
      n_tok))
  if (vec) GO(true);
  else GO(false);
#undef GO
  HY_CHECK();
  return 0;
}

int hy_pair_rows(void* out, int ld_out, const void* proj, int ld, int g_off,
                 const void* cache, const void* pos, const void* row,
                 const void* bt, int max_blocks, int H, int G, int D, int V,
                 const void* q_scale, float cap, float lam, float gain,
                 float eps, int n_rows, int dtype, void* stream) {
  if (G <= 0 || H <= 0 || H % G || H > 65535 || D <= 0 || D > 1024 ||
      V <= 0 || V > 1024)
    return -2;
  if (n_rows <= 0) return 0;
  int cw = 1;
  while (cw < V && cw < 256) cw *= 2;
  const bool vec = D % 4 == 0 && V % 4 == 0;
  const dim3 grid(n_rows, H), block(256);
#define GO(NC)                                                              \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                       \
      (pair_rows_kernel<T, NC>), grid, block,                               \
      (2 * D + 768 + 512 * NC) * sizeof(float), (hipStream_t)stream,        \
      (T*)out, ld_out, (const T*)proj, ld, g_off, (const T*)cache,          \
      (const int*)pos, (const int*)row, (const int*)bt, max_blocks, H, G, D, \
      V, cw, (const float*)q_scale, cap, lam, gain, eps, vec))
  if (V <= 256) GO(1);
  else if (V <= 512) GO(2);
  else GO(4);
#undef GO
  HY_CHECK();
  return 0;
}

}  // extern "C"
