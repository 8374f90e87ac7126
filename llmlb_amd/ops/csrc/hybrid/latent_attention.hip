// Attention over a cache of latents.
//
// A cached token is one row of rank + R numbers: a normed latent c and a
// rotated key part that all heads share.  Head h's key is (W_uk c, kr)
// and its value W_uv c, so with qa = W_uk^T q (the "absorbed" query)
//   score = (qa . c + qr . kr) * scale,   out = W_uv (sum_j p_j c_j):
// the cache is read as it is, once for all heads.  A query at position i
// sees the keys j with 0 <= i - j < window.  With ``sink`` (a number per
// head) the softmax's sum also contains exp(sink), which has no value.
//
// Cache layout: [pages][16 tokens][rank + R].
#include "common.h"

// Per token of a packed batch: norm the latent, rotate the key part and
// put both into the cache; rotate every head's query part in place.
// Column offsets are into a row of ``proj`` (ld columns).  The pair
// (i, i + R/2) turns; cos_sin row p is cos[R/2] | sin[R/2].  One wave a
// token; VQ and VC: query parts and latents come in whole vectors.
template <typename T, bool VQ, bool VC>
__global__ __launch_bounds__(256) void latent_prep_kernel(
    T* __restrict__ proj, int ld, int H, int D, int R, int c_off, int rank,
    const float* __restrict__ w_norm, float eps,
    const float* __restrict__ cos_sin, const int* __restrict__ pos_,
    const int* __restrict__ row_, const int* __restrict__ bt, int max_blocks,
    T* __restrict__ cache, int writes_kv, int n_tok) {
  const int t = blockIdx.x * 4 + threadIdx.x / WAVE;
  if (t >= n_tok) return;
  const int lane = threadIdx.x & (WAVE - 1);
  const int pos = pos_[t];
  T* p = proj + (size_t)t * ld;
  const int half = R / 2;
  const float* cs = cos_sin + (size_t)pos * R;
  // the latent's loads and the page lookup go first: the longest chains
  constexpr int KEEP = 2;
  float keep[KEEP][8], ssq = 0.f;
  const T* src = p + c_off;
  T* dst = nullptr;
  float kr[2] = {0.f, 0.f};
  if (writes_kv) {
    dst = cache + page_slot(bt, max_blocks, row_[t], pos) * (rank + R);
    if (lane < half) {
      kr[0] = to_f(src[rank + lane]);
      kr[1] = to_f(src[rank + half + lane]);
    }
    if (VC) {
#pragma unroll
      for (int n = 0; n < KEEP; ++n) {
        const int i = (lane + n * WAVE) * 8;
        if (i < rank) {
          load8(src + i, keep[n]);
#pragma unroll
          for (int j = 0; j < 8; ++j) ssq += keep[n][j] * keep[n][j];
        }
      }
    }
    for (int i = lane + (VC ? KEEP * WAVE * 8 : 0); i < rank; i += WAVE) {
      const float f = to_f(src[i]);
      ssq += f * f;
    }
  }
  if (VQ) {
    const int quads = half / 4;
    for (int i = lane; i < H * quads; i += WAVE) {
      const int h = i / quads, j = (i - h * quads) * 4;
      T* q = p + (size_t)h * (D + R) + D + j;
      float u[4], v[4];
      load4(q, u);
      load4(q + half, v);
      const float4 c = *reinterpret_cast<const float4*>(cs + j);
      const float4 s = *reinterpret_cast<const float4*>(cs + half + j);
      const float a[4] = {u[0] * c.x - v[0] * s.x, u[1] * c.y - v[1] * s.y,
                          u[2] * c.z - v[2] * s.z, u[3] * c.w - v[3] * s.w};
      const float b[4] = {v[0] * c.x + u[0] * s.x, v[1] * c.y + u[1] * s.y,
                          v[2] * c.z + u[2] * s.z, v[3] * c.w + u[3] * s.w};
      store4(q, a);
      store4(q + half, b);
    }
  } else {
    for (int i = lane; i < H * half; i += WAVE) {
      const int h = i / half, j = i % half;
      T* q = p + (size_t)h * (D + R) + D + j;
      const float u = to_f(q[0]), v = to_f(q[half]);
      const float c = cs[j], s = cs[half + j];
      q[0] = from_f<T>(u * c - v * s);
      q[half] = from_f<T>(v * c + u * s);
    }
  }
  if (!writes_kv) return;
  const float r = 1.f / sqrtf(wave_sum(ssq) / rank + eps);
  if (VC) {
#pragma unroll
    for (int n = 0; n < KEEP; ++n) {
      const int i = (lane + n * WAVE) * 8;
      if (i < rank) {
        float w[8];
        load8(w_norm + i, w);
#pragma unroll
        for (int j = 0; j < 8; ++j) keep[n][j] *= r * w[j];
        store8(dst + i, keep[n]);
      }
    }
  }
  for (int i = lane + (VC ? KEEP * WAVE * 8 : 0); i < rank; i += WAVE)
    dst[i] = from_f<T>(to_f(src[i]) * r * w_norm[i]);
  for (int j = lane; j < half; j += WAVE) {
    const float u = j == lane ? kr[0] : to_f(src[rank + j]);
    const float v = j == lane ? kr[1] : to_f(src[rank + half + j]);
    const float c = cs[j], s = cs[half + j];
    dst[rank + j] = from_f<T>(u * c - v * s);
    dst[rank + half + j] = from_f<T>(v * c + u * s);
  }
}

// Absorbed attention of any sizes, one workgroup per (query, head): the
// waves take every fourth key each and merge at the end.  The 32-bit
// path, and 16-bit sizes that the tiled kernels do not cover.
//   qa  [H][N][rank], proj rows carry the rotated query parts
//   out [H][N][rank]
template <typename T, int NR>
__global__ __launch_bounds__(256) void latent_rows_kernel(
    T* __restrict__ out, const T* __restrict__ qa, const T* __restrict__ proj,
    int ld, int D, int R, int rank, const T* __restrict__ cache,
    const int* __restrict__ pos_, const int* __restrict__ row_,
    const int* __restrict__ bt, int max_blocks, int window, float scale,
    const float* __restrict__ sink, int N) {
  extern __shared__ float lds[];
  float* lq = lds;               // rank + R query numbers
  float* lacc = lds + rank + R;  // 4 waves x rank
  __shared__ float lm[4], ll[4];
  const int n = blockIdx.x, h = blockIdx.y;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const int pos = pos_[n], row = row_[n];
  const int first = pos - window + 1 > 0 ? pos - window + 1 : 0;
  const T* q = qa + ((size_t)h * N + n) * rank;
  for (int i = threadIdx.x; i < rank; i += 256) lq[i] = to_f(q[i]) * scale;
  const T* qr = proj + (size_t)n * ld + (size_t)h * (D + R) + D;
  for (int i = threadIdx.x; i < R; i += 256)
    lq[rank + i] = to_f(qr[i]) * scale;
  __syncthreads();

  float m = -INFINITY, l = 0.f, acc[NR];
  if (sink && wave == 0) {
    m = sink[h];
    l = 1.f;
  }
#pragma unroll
  for (int i = 0; i < NR; ++i) acc[i] = 0.f;
  for (int j = first + wave; j <= pos; j += 4) {
    const T* key = cache + page_slot(bt, max_blocks, row, j) * (rank + R);
    float c[NR], s = 0.f;
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int d = lane + i * WAVE;
      c[i] = d < rank ? to_f(key[d]) : 0.f;
      s += d < rank ? c[i] * lq[d] : 0.f;
    }
    for (int d = lane; d < R; d += WAVE) s += to_f(key[rank + d]) * lq[rank + d];
    s = wave_sum(s);
    const float mn = fmaxf(m, s);
    const float keep = expf(m - mn), w = expf(s - mn);
    l = l * keep + w;
#pragma unroll
    for (int i = 0; i < NR; ++i) acc[i] = acc[i] * keep + w * c[i];
    m = mn;
  }
  if (lane == 0) {
    lm[wave] = m;
    ll[wave] = l;
  }
#pragma unroll
  for (int i = 0; i < NR; ++i)
    if (lane + i * WAVE < rank) lacc[wave * rank + lane + i * WAVE] = acc[i];
  __syncthreads();
  const float mx = fmaxf(fmaxf(lm[0], lm[1]), fmaxf(lm[2], lm[3]));
  float f[4], sum = 0.f;
#pragma unroll
  for (int w = 0; w < 4; ++w) {
    f[w] = ll[w] > 0.f ? expf(lm[w] - mx) : 0.f;
    sum += f[w] * ll[w];
  }
  const float inv = 1.f / sum;
  T* o = out + ((size_t)h * N + n) * rank;
  for (int i = threadIdx.x; i < rank; i += 256) {
    float v = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) v += f[w] * lacc[w * rank + i];
    o[i] = from_f<T>(v * inv);
  }
}

// out[t][h V ..] = o[h][t][..] sigmoid(gate[t][h V ..]), the absorbed
// form's values side by side.  N columns a thread.
template <typename T, int N>
__global__ __launch_bounds__(256) void join_heads_kernel(
    T* __restrict__ out, const T* __restrict__ o, const T* __restrict__ gate,
    int ld, int n_tok, int H, int V) {
  const int per = V / N;
  const long long id = (long long)blockIdx.x * 256 + threadIdx.x;
  if (id >= (long long)n_tok * H * per) return;
  const int c = (int)(id % per) * N;
  const long long th = id / per;
  const int t = (int)(th / H), h = (int)(th - (long long)t * H);
  const T* src = o + ((size_t)h * n_tok + t) * V + c;
  const T* g = gate + (size_t)t * ld + (size_t)h * V + c;
  T* dst = out + ((size_t)t * H + h) * V + c;
  float f[N], z[N];
  if constexpr (N == 8) {
    load8(src, f);
    load8(g, z);
  } else {
    f[0] = to_f(src[0]);
    z[0] = to_f(g[0]);
  }
#pragma unroll
  for (int i = 0; i < N; ++i) f[i] *= sigmoid_f(z[i]);
  if constexpr (N == 8) store8(dst, f);
  else dst[0] = from_f<T>(f[0]);
}

extern "C" {

int hy_join_heads(void* out, const void* o, const void* gate, int ld,
                  int n_tok, int H, int V, int dtype, void* stream) {
  if (H <= 0 || V <= 0) return -2;
  if (n_tok <= 0) return 0;
  const uintptr_t mask = dtype == 0 ? 15 : 31;
  const bool vec = V % 8 == 0 && ld % 8 == 0 &&
                   (((uintptr_t)out | (uintptr_t)o | (uintptr_t)gate) &
                    mask) == 0;
  const long long n = (long long)n_tok * H * (V / (vec ? 8 : 1));
  if (n >= (1ll << 38)) return -2;
  const dim3 grid((unsigned)((n + 255) / 256)), block(256);
#define GO(N)                                                              \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                      \
      (join_heads_kernel<T, N>), grid, block, 0, (hipStream_t)stream,      \
      (T*)out, (const T*)o, (const T*)gate, ld, n_tok, H, V))
  if (vec) GO(8);
  else GO(1);
#undef GO
  HY_CHECK();
  return 0;
}

int hy_latent_prep(void* proj, int ld, int H, int D, int R, int c_off,
                   int rank, const void* w_norm, float eps,
                   const void* cos_sin, const void* pos, const void* row,
                   const void* bt, int max_blocks, void* cache, int writes_kv,
                   int n_tok, int dtype, void* stream) {
  if (R % 2 || rank <= 0) return -2;
  if (n_tok <= 0) return 0;
  const bool vq = R % 8 == 0 && D % 4 == 0 && ld % 4 == 0;
  const bool vc = rank % 8 == 0 && R % 8 == 0 && ld % 8 == 0 &&
                  c_off % 8 == 0;
#define GO(VQ, VC)                                                           \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                        \
      (latent_prep_kernel<T, VQ, VC>), dim3((n_tok + 3) / 4), dim3(256), 0,  \
      (hipStream_t)stream, (T*)proj, ld, H, D, R, c_off, rank,               \
      (const float*)w_norm, eps, (const float*)cos_sin, (const int*)pos,     \
      (const int*)row, (const int*)bt, max_blocks, (T*)cache, writes_kv,     \
      n_tok))
  if (vq && vc) GO(true, true);
  else if (vq) GO(true, false);
  else if (vc) GO(false, true);
  else GO(false, false);
#undef GO
  HY_CHECK();
  return 0;
}

int hy_latent_rows(void* out, const void* qa, const void* proj, int ld, int H,
                   int D, int R, int rank, const void* cache, const void* pos,
                   const void* row, const void* bt, int max_blocks,
                   int window, float scale, const void* sink, int n_rows,
                   int dtype, void* stream) {
  if (rank <= 0 || rank > 2048 || R > 2048 || window <= 0 || H > 65535)
    return -2;
  if (n_rows <= 0) return 0;
  const size_t lds = (size_t)(5 * rank + R) * sizeof(float);
  const dim3 grid(n_rows, H), block(256);
#define GO(NR)                                                               \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                        \
      (latent_rows_kernel<T, NR>), grid, block, lds, (hipStream_t)stream,    \
      (T*)out, (const T*)qa, (const T*)proj, ld, D, R, rank,                 \
      (const T*)cache, (const int*)pos, (const int*)row, (const int*)bt,     \
      max_blocks, window, scale, (const float*)sink, n_rows))
  if (rank <= 128) GO(2);
  else if (rank <= 256) GO(4);
  else if (rank <= 512) GO(8);
  else if (rank <= 1024) GO(16);
  else GO(32);
#undef GO
  HY_CHECK();
  return 0;
}

}  // extern "C"
