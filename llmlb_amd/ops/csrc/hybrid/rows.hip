// Row and elementwise kernels of the hybrid models: a residual stream
// in 32-bit, an RMS norm applied to a sublayer's OUTPUT, the tanh form
// of gelu and the soft cap of the logits.
#include "common.h"

// x[t] = table[ids[t]] in 32-bit, and a copy in the storage type for the
// first projection (null when the storage type is float).
template <typename T>
__global__ __launch_bounds__(256) void embed_rows_kernel(
    float* __restrict__ x, T* __restrict__ xb, const T* __restrict__ table,
    const int* __restrict__ ids, int width, int vocab) {
  const int t = blockIdx.x;
  const int id = ids[t];
  const bool ok = id >= 0 && id < vocab;
  const T* src = table + (size_t)(ok ? id : 0) * width;
  if (ok && (width & 7) == 0) {
    for (int i = threadIdx.x * 8; i < width; i += 2048) {
      float f[8];
      load8(src + i, f);
      store8(x + (size_t)t * width + i, f);
      if (xb) store8(xb + (size_t)t * width + i, f);
    }
    return;
  }
  for (int i = threadIdx.x; i < width; i += 256) {
    const float v = ok ? to_f(src[i]) : 0.f;
    x[(size_t)t * width + i] = v;
    if (xb) xb[(size_t)t * width + i] = from_f<T>(v);
  }
}

// x += y / sqrt(mean(y^2) + eps) * (w_offset + w); xb = x in the storage
// type.  One workgroup per row; up to 4 vectors a thread stay in
// registers between the two passes, the rest is read again.
#define NORM_KEEP 4
template <typename T>
__global__ __launch_bounds__(256) void post_norm_add_kernel(
    float* __restrict__ x, T* __restrict__ xb, const T* __restrict__ y,
    const float* __restrict__ w, float w_offset, int width, float eps) {
  __shared__ float red[4];
  const size_t base = (size_t)blockIdx.x * width;
  const bool vec = (width & 7) == 0;
  const int nvec = vec ? width >> 3 : 0;
  float keep[NORM_KEEP][8];
  float ssq = 0.f;
#pragma unroll
  for (int n = 0; n < NORM_KEEP; ++n) {
    const int i = threadIdx.x + n * 256;
    if (i < nvec) {
      load8(y + base + i * 8, keep[n]);
#pragma unroll
      for (int j = 0; j < 8; ++j) ssq += keep[n][j] * keep[n][j];
    }
  }
  for (int i = threadIdx.x + NORM_KEEP * 256; i < nvec; i += 256) {
    float f[8];
    load8(y + base + i * 8, f);
#pragma unroll
    for (int j = 0; j < 8; ++j) ssq += f[j] * f[j];
  }
  if (!vec)
    for (int i = threadIdx.x; i < width; i += 256) {
      const float f = to_f(y[base + i]);
      ssq += f * f;
    }
  const float r = 1.f / sqrtf(block_sum_256(ssq, red) / width + eps);

  auto emit = [&](int i, const float* f) {
    float xr[8], wr[8];
    load8(x + base + i * 8, xr);
    load8(w + i * 8, wr);
#pragma unroll
    for (int j = 0; j < 8; ++j) xr[j] += f[j] * r * (w_offset + wr[j]);
    store8(x + base + i * 8, xr);
    if (xb) store8(xb + base + i * 8, xr);
  };
#pragma unroll
  for (int n = 0; n < NORM_KEEP; ++n) {
    const int i = threadIdx.x + n * 256;
    if (i < nvec) emit(i, keep[n]);
  }
  for (int i = threadIdx.x + NORM_KEEP * 256; i < nvec; i += 256) {
    float f[8];
    load8(y + base + i * 8, f);
    emit(i, f);
  }
  if (!vec)
    for (int i = threadIdx.x; i < width; i += 256) {
      const float v =
          x[base + i] + to_f(y[base + i]) * r * (w_offset + w[i]);
      x[base + i] = v;
      if (xb) xb[base + i] = from_f<T>(v);
    }
}

// out[r] = norm(x[index[r]]) in the storage type (index null: row r).
template <typename T>
__global__ __launch_bounds__(256) void norm_rows_kernel(
    T* __restrict__ out, const float* __restrict__ x,
    const int* __restrict__ index, const float* __restrict__ w,
    float w_offset, int width, float eps) {
  __shared__ float red[4];
  const size_t src = (size_t)(index ? index[blockIdx.x] : blockIdx.x) * width;
  const size_t dst = (size_t)blockIdx.x * width;
  float ssq = 0.f;
  if ((width & 7) == 0) {
    for (int i = threadIdx.x * 8; i < width; i += 2048) {
      float f[8];
      load8(x + src + i, f);
#pragma unroll
      for (int j = 0; j < 8; ++j) ssq += f[j] * f[j];
    }
    const float r = 1.f / sqrtf(block_sum_256(ssq, red) / width + eps);
    for (int i = threadIdx.x * 8; i < width; i += 2048) {
      float f[8], wr[8];
      load8(x + src + i, f);
      load8(w + i, wr);
#pragma unroll
      for (int j = 0; j < 8; ++j) f[j] *= r * (w_offset + wr[j]);
      store8(out + dst + i, f);
    }
    return;
  }
  for (int i = threadIdx.x; i < width; i += 256)
    ssq += x[src + i] * x[src + i];
  const float r = 1.f / sqrtf(block_sum_256(ssq, red) / width + eps);
  for (int i = threadIdx.x; i < width; i += 256)
    out[dst + i] = from_f<T>(x[src + i] * r * (w_offset + w[i]));
}

__device__ __forceinline__ float gelu_tanh_f(float z) {
  const float k = 0.7978845608028654f;  // sqrt(2 / pi)
  return 0.5f * z * (1.f + tanhf(k * (z + 0.044715f * z * z * z)));
}
// the same through one exponential, for 16-bit results
__device__ __forceinline__ float gelu_tanh_fast(float z) {
  const float k = 0.7978845608028654f;
  const float t = k * (z + 0.044715f * z * z * z);
  return z / (1.f + __expf(-2.f * t));
}

template <typename T>
__global__ __launch_bounds__(256) void gelu_tanh_kernel(T* __restrict__ y,
                                                        long long n) {
  const long long nvec = n >> 3;
  const long long id = (long long)blockIdx.x * 256 + threadIdx.x;
  const long long step = (long long)gridDim.x * 256;
  for (long long i = id; i < nvec; i += step) {
    float f[8];
    load8(y + i * 8, f);
#pragma unroll
    for (int j = 0; j < 8; ++j)
      f[j] = sizeof(T) == 2 ? gelu_tanh_fast(f[j]) : gelu_tanh_f(f[j]);
    store8(y + i * 8, f);
  }
  for (long long i = nvec * 8 + id; i < n; i += step)
    y[i] = from_f<T>(gelu_tanh_f(to_f(y[i])));
}

// out = cap * tanh(in / cap) in 32-bit (cap <= 0: a plain widening)
template <typename T>
__global__ __launch_bounds__(256) void soft_cap_kernel(
    float* __restrict__ out, const T* __restrict__ in, float cap,
    long long n) {
  const long long step = (long long)gridDim.x * 256;
  const long long id = (long long)blockIdx.x * 256 + threadIdx.x;
  const long long nvec = n >> 3;
  for (long long i = id; i < nvec; i += step) {
    float f[8];
    load8(in + i * 8, f);
    if (cap > 0.f) {
#pragma unroll
      for (int j = 0; j < 8; ++j) f[j] = cap * tanhf(f[j] / cap);
    }
    store8(out + i * 8, f);
  }
  for (long long i = nvec * 8 + id; i < n; i += step) {
    const float v = to_f(in[i]);
    out[i] = cap > 0.f ? cap * tanhf(v / cap) : v;
  }
}

extern "C" {

int hy_embed_rows(void* x, void* xb, const void* table, const void* ids,
                  int n_tok, int width, int vocab, int dtype, void* stream) {
  if (n_tok <= 0) return 0;
  HY_DTYPE(dtype, hipLaunchKernelGGL(
      embed_rows_kernel<T>, dim3(n_tok), dim3(256), 0, (hipStream_t)stream,
      (float*)x, (T*)xb, (const T*)table, (const int*)ids, width, vocab));
  HY_CHECK();
  return 0;
}

int hy_post_norm_add(void* x, void* xb, const void* y, const void* w,
                     float w_offset, int n_tok, int width, float eps,
                     int dtype, void* stream) {
  if (n_tok <= 0) return 0;
  HY_DTYPE(dtype, hipLaunchKernelGGL(
      post_norm_add_kernel<T>, dim3(n_tok), dim3(256), 0,
      (hipStream_t)stream, (float*)x, (T*)xb, (const T*)y, (const float*)w,
      w_offset, width, eps));
  HY_CHECK();
  return 0;
}

int hy_norm_rows(void* out, const void* x, const void* index, const void* w,
                 float w_offset, int n_rows, int width, float eps, int dtype,
                 void* stream) {
  if (n_rows <= 0) return 0;
  HY_DTYPE(dtype, hipLaunchKernelGGL(
      norm_rows_kernel<T>, dim3(n_rows), dim3(256), 0, (hipStream_t)stream,
      (T*)out, (const float*)x, (const int*)index, (const float*)w, w_offset,
      width, eps));
  HY_CHECK();
  return 0;
}

static int grid_for(long long items) {
  long long g = (items + 255) / 256;
  return (int)(g < 1 ? 1 : (g > 8192 ? 8192 : g));
}

int hy_gelu_tanh(void* y, long long n, int dtype, void* stream) {
  if (n <= 0) return 0;
  HY_DTYPE(dtype, hipLaunchKernelGGL(
      gelu_tanh_kernel<T>, dim3(grid_for((n + 7) / 8)), dim3(256), 0,
      (hipStream_t)stream, (T*)y, n));
  HY_CHECK();
  return 0;
}

int hy_soft_cap(void* out, const void* in, float cap, long long n, int dtype,
                void* stream) {
  if (n <= 0) return 0;
  HY_DTYPE(dtype, hipLaunchKernelGGL(
      soft_cap_kernel<T>, dim3(grid_for((n + 7) / 8)), dim3(256), 0,
      (hipStream_t)stream, (float*)out, (const T*)in, cap, n));
  HY_CHECK();
  return 0;
}

}  // extern "C"
