// Queries and keys of attention whose heads are normed one by one: biases
// added, each head divided by its root mean square, weighted (one weight
// for all heads of a kind), rotated on its first ``rot`` numbers, the
// pair (i, i + rot / 2) turning together.  Queries stay in their row of
// the projection; keys and values go into the pages of window_attention.hip.
// Without values of their own (v_off < 0) the values are the keys with
// their biases, before norm and rotation.
#include "common.h"

struct HeadPrep {
  void* proj;   // [n_tok][ld]: queries first, keys (and values) at offsets
  void* cache;
  const float* bq;  // [H D], [G D]; null: none
  const float* bk;
  const float* wq;  // [D]
  const float* wk;
  const float* cos_sin;  // [positions][rot], cosines first
  const int* pos;
  const int* row;
  const int* bt;
  int ld, k_off, v_off, H, G, D, V, rot, max_blocks, n_tok;
  float eps;
};

// place of a key/value head's cached row
template <typename T>
__device__ __forceinline__ T* cached_row(const HeadPrep& a, int t, int pos,
                                         int g) {
  const int page = a.bt[(size_t)a.row[t] * a.max_blocks + pos / PAGE];
  return (T*)a.cache +
         (((size_t)page * a.G + g) * PAGE + pos % PAGE) * (a.D + a.V);
}

// L lanes a head, each with two pieces of 8: a piece and the one it is
// rotated with, or two neighbours past the rotated part.
template <typename T>
__global__ __launch_bounds__(256) void head_prep_kernel(HeadPrep a, int L) {
  const int D = a.D, rot = a.rot;
  const int heads = a.H + a.G;
  const long long unit =
      ((long long)blockIdx.x * 256 + threadIdx.x) / L;
  if (unit >= (long long)a.n_tok * heads) return;  // whole groups of L
  const int lane = threadIdx.x % L;
  const int t = (int)(unit / heads), hd = (int)(unit - (long long)t * heads);
  const bool key = hd >= a.H;
  const int g = hd - a.H;
  const bool used = lane < D / 16;
  const int i = used ? lane : 0;
  const bool turned = i < rot / 16;
  const int d = turned ? i * 8 : rot + (i - rot / 16) * 16;
  const int e = d + (turned ? rot / 2 : 8);
  T* src = (T*)a.proj + (size_t)t * a.ld +
           (key ? a.k_off + g * D : hd * D);
  const int pos = a.pos[t];
  float lo[8], hi[8], c[8], s[8];
  load8(src + d, lo);
  load8(src + e, hi);
  if (turned) {
    const float* cs = a.cos_sin + (size_t)pos * rot;
    load8(cs + d, c);
    load8(cs + rot / 2 + d, s);
  }
  const float* bias = key ? a.bk : a.bq;
  if (bias) {
    bias += key ? g * D : hd * D;
    float f[8];
    load8(bias + d, f);
#pragma unroll
    for (int j = 0; j < 8; ++j) lo[j] += f[j];
    load8(bias + e, f);
#pragma unroll
    for (int j = 0; j < 8; ++j) hi[j] += f[j];
  }
  float ssq = 0.f;
#pragma unroll
  for (int j = 0; j < 8; ++j) ssq += lo[j] * lo[j] + hi[j] * hi[j];
  if (!used) ssq = 0.f;
  for (int o = L / 2; o > 0; o >>= 1) ssq += __shfl_xor(ssq, o, WAVE);
  T* dst = src;
  if (key) {
    dst = cached_row<T>(a, t, pos, g);
    if (a.v_off < 0) {
      if (used) {
        store8(dst + D + d, lo);
        store8(dst + D + e, hi);
      }
    } else {
      const T* v = (const T*)a.proj + (size_t)t * a.ld + a.v_off + g * a.V;
      for (int j = lane * 8; j < a.V; j += L * 8) {
        float f[8];
        load8(v + j, f);
        store8(dst + D + j, f);
      }
    }
  }
  if (!used) return;
  const float r = 1.f / sqrtf(ssq / D + a.eps);
  const float* w = key ? a.wk : a.wq;
  float f[8];
  load8(w + d, f);
#pragma unroll
  for (int j = 0; j < 8; ++j) lo[j] *= r * f[j];
  load8(w + e, f);
#pragma unroll
  for (int j = 0; j < 8; ++j) hi[j] *= r * f[j];
  if (turned) {
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const float x = lo[j];
      lo[j] = x * c[j] - hi[j] * s[j];
      hi[j] = hi[j] * c[j] + x * s[j];
    }
  }
  store8(dst + d, lo);
  store8(dst + e, hi);
}

// Any sizes: a wave a head, its numbers through LDS.
template <typename T>
__global__ __launch_bounds__(256) void head_prep_any_kernel(HeadPrep a) {
  extern __shared__ float lds[];
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const int D = a.D, rot = a.rot, half = rot / 2;
  const int t = blockIdx.x, hd = blockIdx.y * 4 + wave;
  const bool real = hd < a.H + a.G;
  const bool key = hd >= a.H;
  const int g = hd - a.H;
  float* x = lds + wave * D;
  const int pos = a.pos[t];
  T* src = (T*)a.proj + (size_t)t * a.ld +
           (key ? a.k_off + (real ? g : 0) * D : hd * D);
  T* dst = src;
  float r = 0.f;
  if (real) {
    const float* bias = key ? a.bk : a.bq;
    if (bias) bias += key ? g * D : hd * D;
    if (key) dst = cached_row<T>(a, t, pos, g);
    float ssq = 0.f;
    for (int d = lane; d < D; d += WAVE) {
      const float f = to_f(src[d]) + (bias ? bias[d] : 0.f);
      ssq += f * f;
      x[d] = f;
      if (key && a.v_off < 0) dst[D + d] = from_f<T>(f);
    }
    if (key && a.v_off >= 0) {
      const T* v = (const T*)a.proj + (size_t)t * a.ld + a.v_off + g * a.V;
      for (int d = lane; d < a.V; d += WAVE) dst[D + d] = v[d];
    }
    r = 1.f / sqrtf(wave_sum(ssq) / D + a.eps);
  }
  __syncthreads();
  if (!real) return;
  const float* w = key ? a.wk : a.wq;
  const float* cs = a.cos_sin + (size_t)pos * rot;
  for (int d = lane; d < D; d += WAVE) {
    float f = x[d] * r * w[d];
    if (d < half)
      f = f * cs[d] - x[d + half] * r * w[d + half] * cs[half + d];
    else if (d < rot)
      f = f * cs[d - half] + x[d - half] * r * w[d - half] * cs[d];
    dst[d] = from_f<T>(f);
  }
}

extern "C" {

int hy_head_prep(void* proj, int ld, void* cache, int k_off, int v_off, int H,
                 int G, int D, int V, int rot, const void* bq, const void* bk,
                 const void* wq, const void* wk, const void* cos_sin,
                 float eps, const void* pos, const void* row, const void* bt,
                 int max_blocks, int n_tok, int dtype, void* stream) {
  const HeadPrep a{proj,
                   cache,
                   (const float*)bq,
                   (const float*)bk,
                   (const float*)wq,
                   (const float*)wk,
                   (const float*)cos_sin,
                   (const int*)pos,
                   (const int*)row,
                   (const int*)bt,
                   ld, k_off, v_off, H, G, D, V, rot, max_blocks, n_tok,
                   eps};
  if (H <= 0 || G <= 0 || D <= 0 || D > 2048 || V <= 0 || rot < 0 ||
      rot > D || rot % 2 || (rot && !cos_sin) || (v_off < 0 && V != D) ||
      H + G > 65535)
    return -2;
  if (n_tok <= 0) return 0;
  if (D % 16 == 0 && D <= 1024 && rot % 16 == 0 && V % 8 == 0 &&
      ld % 8 == 0 && k_off % 8 == 0 && (v_off < 0 || v_off % 8 == 0)) {
    int L = 1;
    while (L * 16 < D) L *= 2;
    const long long blocks =
        ((long long)n_tok * (H + G) * L + 255) / 256;
    if (blocks >= (1ll << 31)) return -2;
    HY_DTYPE(dtype, hipLaunchKernelGGL(
        head_prep_kernel<T>, dim3((unsigned)blocks), dim3(256), 0,
        (hipStream_t)stream, a, L));
  } else {
    HY_DTYPE(dtype, hipLaunchKernelGGL(
        head_prep_any_kernel<T>, dim3(n_tok, (H + G + 3) / 4), dim3(256),
        4 * D * sizeof(float), (hipStream_t)stream, a));
  }
  HY_CHECK();
  return 0;
}

}  // extern "C"
