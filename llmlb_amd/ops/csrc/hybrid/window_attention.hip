// Grouped-query attention over a sliding window of cached tokens, or over
// the tokens of the query's own chunk (chunks are counted from position
// 0), each head's output times the sigmoid of a number of its own (column
// g_off of its token's row; g_off < 0: no gate).
//
// Queries and keys are prepared by window_prep (normed over the whole
// projection, all heads at once) or by head_prep (each head by itself),
// and rotated on the first ``rot`` numbers of each head.  A cached
// token keeps, for each of G key/value heads, one row [key (D) | value
// (V)]; a page is [G][16 tokens][D + V].  Query head h reads key/value
// head h / (H / G).  The query's weights carry the scale of the scores
// and log2(e): the softmax is over powers of two.
#include "window_prep.h"

// Four tokens a workgroup, a wave each.
template <int KQ, int KK>
__global__ __launch_bounds__(256) void window_prep_wave_kernel(WindowPrep a) {
  const int t =
      blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
  if (t < a.n_tok) window_prep_wave<bf16_t, KQ, KK>(a, t);
}

// Any sizes, a workgroup a token: the section's normed numbers go through LDS.
template <typename T>
__global__ __launch_bounds__(256) void window_prep_kernel(WindowPrep a) {
  extern __shared__ float lds[];
  __shared__ float red[2][4];
  const int t = blockIdx.x, tid = threadIdx.x;
  const int pos = a.pos[t], G = a.G, D = a.D, V = a.V, rot = a.rot;
  T* src = (T*)a.proj + (size_t)t * a.ld;
  const int page = a.bt[(size_t)a.row[t] * a.max_blocks + pos / PAGE];
  T* rows = (T*)a.cache + ((size_t)page * G * PAGE + pos % PAGE) * (D + V);
  const size_t head_step = (size_t)PAGE * (D + V);
  const int half = rot / 2;
  const float* cs = a.cos_sin + (size_t)pos * rot;
  for (int i = tid; i < G * V; i += 256)
    rows[i / V * head_step + D + i % V] = src[a.v_off + i];
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    const int off = s == 0 ? 0 : a.k_off;
    const float* w = s == 0 ? a.wq : a.wk;
    const int n = (s == 0 ? a.H : G) * D;
    float ssq = 0.f;
    for (int i = tid; i < n; i += 256) {
      const float x = to_f(src[off + i]);
      ssq += x * x;
    }
    const float r = 1.f / sqrtf(block_sum_256(ssq, red[s]) / n + a.eps);
    for (int i = tid; i < n; i += 256)
      lds[i] = to_f(src[off + i]) * r * w[i];
    __syncthreads();
    for (int i = tid; i < n; i += 256) {
      const int d = i % D;
      float x = lds[i];
      if (d < half) x = x * cs[d] - lds[i + half] * cs[half + d];
      else if (d < rot) x = x * cs[d - half] + lds[i - half] * cs[d];
      T* dst = s == 0 ? src + off + i : rows + i / D * head_step + d;
      *dst = from_f<T>(x);
    }
    __syncthreads();
  }
}

// Any sizes, 32-bit arithmetic: one workgroup per (query, head).  256 keys
// at a time, a thread scores one of them; then CW threads take the value
// columns of every (256 / CW)th key each.
template <typename T, int NC>
__global__ __launch_bounds__(256) void window_rows_kernel(
    T* __restrict__ out, int ld_out, const T* __restrict__ proj, int ld,
    int g_off, const T* __restrict__ cache, const int* __restrict__ pos_,
    const int* __restrict__ row_, const int* __restrict__ bt, int max_blocks,
    int H, int G, int D, int V, int CW, Mask mask, bool vec) {
  extern __shared__ float lds[];
  float* lq = lds;                     // D query numbers
  float* lp = lq + D;                  // weights of 256 keys
  int* lrow = (int*)(lp + 256);        // rows of the keys
  float* lacc = (float*)(lrow + 256);  // 256 x NC
  __shared__ float red[4], red2[4];
  const int t = blockIdx.x, h = blockIdx.y, g = h / (H / G);
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & (WAVE - 1);
  const int pos = pos_[t];
  const int* pages = bt + (size_t)row_[t] * max_blocks;
  const int width = D + V;
  const T* q = proj + (size_t)t * ld + (size_t)h * D;
  for (int i = tid; i < D; i += 256) lq[i] = to_f(q[i]);
  const int grp = tid / CW, ngrp = 256 / CW, c0 = tid % CW;
  float m = -INFINITY, l = 0.f, acc[NC];
#pragma unroll
  for (int i = 0; i < NC; ++i) acc[i] = 0.f;
  __syncthreads();
  for (int j0 = mask.first(pos); j0 <= pos; j0 += 256) {
    const int j = j0 + tid;
    float s = -INFINITY;
    if (j <= pos) {
      const int row = (pages[j / PAGE] * G + g) * PAGE + j % PAGE;
      lrow[tid] = row;
      const T* k = cache + (size_t)row * width;
      float a = 0.f;
      if (vec) {
        for (int d = 0; d < D; d += 4) {
          float f[4];
          load4(k + d, f);
#pragma unroll
          for (int i = 0; i < 4; ++i) a += f[i] * lq[d + i];
        }
      } else {
        for (int d = 0; d < D; ++d) a += to_f(k[d]) * lq[d];
      }
      s = a;
    }
    float x = s;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) x = fmaxf(x, __shfl_xor(x, o, WAVE));
    if (lane == 0) red[wave] = x;
    __syncthreads();
    x = fmaxf(fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])), m);
    const float keep = exp2f(m - x);
    m = x;
    const float p = exp2f(s - x);
    l = l * keep + p;
    lp[tid] = p;
    __syncthreads();
    const int n_keys = pos - j0 + 1 < 256 ? pos - j0 + 1 : 256;
#pragma unroll
    for (int i = 0; i < NC; ++i) acc[i] *= keep;
    for (int k = grp; k < n_keys; k += ngrp) {
      const T* v = cache + (size_t)lrow[k] * width + D;
#pragma unroll
      for (int i = 0; i < NC; ++i) {
        const int c = c0 + i * CW;
        acc[i] += lp[k] * (c < V ? to_f(v[c]) : 0.f);
      }
    }
    __syncthreads();
  }
  l = wave_sum(l);
  if (lane == 0) red2[wave] = l;
#pragma unroll
  for (int i = 0; i < NC; ++i) lacc[i * 256 + tid] = acc[i];
  __syncthreads();
  if (grp != 0) return;
  const float gate =
      g_off < 0 ? 1.f : sigmoid_f(to_f(proj[(size_t)t * ld + g_off + h]));
  const float f = gate / (red2[0] + red2[1] + red2[2] + red2[3]);
  T* dst = out + (size_t)t * ld_out + (size_t)h * V;
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = c0 + i * CW;
    float a = 0.f;
    for (int k = 0; k < ngrp; ++k) a += lacc[i * 256 + k * CW + c0];
    if (c < V) dst[c] = from_f<T>(a * f);
  }
}

extern "C" {

int hy_window_prep(void* proj, int ld, void* cache, int k_off, int v_off,
                   int H, int G, int D, int V, int rot, const void* wq,
                   const void* wk, const void* cos_sin, float eps,
                   const void* pos, const void* row, const void* bt,
                   int max_blocks, int n_tok, int dtype, void* stream) {
  const WindowPrep a{proj,
                     cache,
                     (const float*)wq,
                     (const float*)wk,
                     (const float*)cos_sin,
                     (const int*)pos,
                     (const int*)row,
                     (const int*)bt,
                     ld, k_off, v_off, H, G, D, V, rot, max_blocks, n_tok,
                     eps};
  if (!window_prep_ok(a)) return -2;
  if (n_tok <= 0) return 0;
  if (dtype == 0 && window_prep_wave_ok(a)) {
#define GO(KQ, KK)                                                        \
  hipLaunchKernelGGL((window_prep_wave_kernel<KQ, KK>),                   \
                     dim3((n_tok + 3) / 4), dim3(256), 0,                 \
                     (hipStream_t)stream, a)
    WINDOW_PREP_UNITS(H * D, G * D);
#undef GO
  } else {
    HY_DTYPE(dtype, hipLaunchKernelGGL(
        window_prep_kernel<T>, dim3(n_tok), dim3(256),
        (H > G ? H : G) * D * sizeof(float), (hipStream_t)stream, a));
  }
  HY_CHECK();
  return 0;
}

int hy_window_rows(void* out, int ld_out, const void* proj, int ld, int g_off,
                   const void* cache, const void* pos, const void* row,
                   const void* bt, int max_blocks, int H, int G, int D, int V,
                   int window, int chunk, int n_rows, int dtype,
                   void* stream) {
  if (G <= 0 || H <= 0 || H % G || H > 65535 || D <= 0 || D > 1024 ||
      V <= 0 || V > 1024 || window < 1)
    return -2;
  if (n_rows <= 0) return 0;
  int cw = 1;
  while (cw < V && cw < 256) cw *= 2;
  const bool vec = D % 4 == 0 && V % 4 == 0;
  const Mask mask{window, chunk != 0};
  const dim3 grid(n_rows, H), block(256);
#define GO(NC)                                                              \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                       \
      (window_rows_kernel<T, NC>), grid, block,                             \
      (D + 512 + 256 * NC) * sizeof(float), (hipStream_t)stream, (T*)out,   \
      ld_out, (const T*)proj, ld, g_off, (const T*)cache, (const int*)pos,  \
      (const int*)row, (const int*)bt, max_blocks, H, G, D, V, cw, mask,    \
      vec))
  if (V <= 256) GO(1);
  else if (V <= 512) GO(2);
  else GO(4);
#undef GO
  HY_CHECK();
  return 0;
}

}  // extern "C"
