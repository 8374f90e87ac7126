// Row and elementwise kernels of the hybrid models: a residual stream
// in 32-bit, RMS and layer norms of a sublayer's OUTPUT or of the stream
// itself, gated norms of parts of a row, activations, the soft cap of
// logits.
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

// x += mult y; h1 = x / rms(x) * w1, h2 = x / rms(x) * w2 in the storage
// type.  y null: nothing is added; w2 (and h2) null: one norm; w1 null: the
// sum alone.  ROUTED: x += mult (y + sum over k of zw[k] z[k]) with ``top``
// more rows z of the token.  ONE: w1 and w2 are single numbers.  One
// workgroup per row, kept in registers between the passes where it fits.
template <typename T, bool ROUTED, bool ONE>
__global__ __launch_bounds__(256) void add_norms_kernel(
    float* __restrict__ x, const T* __restrict__ y,
    const T* __restrict__ z, const float* __restrict__ zw, int top,
    float mult, const float* __restrict__ w1, const float* __restrict__ w2,
    T* __restrict__ h1, T* __restrict__ h2, int width, float eps) {
  __shared__ float red[4];
  const size_t base = (size_t)blockIdx.x * width;
  if (ROUTED) {
    z += base * top;
    zw += (size_t)blockIdx.x * top;
  }
  const bool vec = (width & 7) == 0;
  const int nvec = vec ? width >> 3 : 0;
  float keep[NORM_KEEP][8];
  float ssq = 0.f;
  auto sum = [&](int i, float* f) {
    load8(x + base + i * 8, f);
    if (y) {
      float d[8];
      load8(y + base + i * 8, d);
      if (ROUTED) {
#pragma unroll 4
        for (int k = 0; k < top; ++k) {
          const float g = zw[k];
          float e[8];
          load8(z + (size_t)k * width + i * 8, e);
#pragma unroll
          for (int j = 0; j < 8; ++j) d[j] += g * e[j];
        }
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) f[j] += mult * d[j];
      store8(x + base + i * 8, f);
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) ssq += f[j] * f[j];
  };
#pragma unroll
  for (int n = 0; n < NORM_KEEP; ++n) {
    const int i = threadIdx.x + n * 256;
    if (i < nvec) sum(i, keep[n]);
  }
  for (int i = threadIdx.x + NORM_KEEP * 256; i < nvec; i += 256) {
    float f[8];
    sum(i, f);
  }
  if (!vec)
    for (int i = threadIdx.x; i < width; i += 256) {
      float v = x[base + i];
      if (y) {
        float d = to_f(y[base + i]);
        if (ROUTED)
          for (int k = 0; k < top; ++k)
            d += zw[k] * to_f(z[(size_t)k * width + i]);
        v += mult * d;
        x[base + i] = v;
      }
      ssq += v * v;
    }
  if (!w1) return;
  const float r = 1.f / sqrtf(block_sum_256(ssq, red) / width + eps);

  auto emit = [&](int i, const float* f) {
    float w[8], o[8];
    if (!ONE) load8(w1 + i * 8, w);
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = f[j] * r * (ONE ? w1[0] : w[j]);
    store8(h1 + base + i * 8, o);
    if (!w2) return;
    if (!ONE) load8(w2 + i * 8, w);
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = f[j] * r * (ONE ? w2[0] : w[j]);
    store8(h2 + base + i * 8, o);
  };
#pragma unroll
  for (int n = 0; n < NORM_KEEP; ++n) {
    const int i = threadIdx.x + n * 256;
    if (i < nvec) emit(i, keep[n]);
  }
  // a thread reads back only what it wrote itself
  for (int i = threadIdx.x + NORM_KEEP * 256; i < nvec; i += 256) {
    float f[8];
    load8(x + base + i * 8, f);
    emit(i, f);
  }
  if (!vec)
    for (int i = threadIdx.x; i < width; i += 256) {
      const float v = x[base + i] * r;
      h1[base + i] = from_f<T>(v * w1[ONE ? 0 : i]);
      if (w2) h2[base + i] = from_f<T>(v * w2[ONE ? 0 : i]);
    }
}

// Each of a row's ``groups`` parts of S columns divided by its rms, times
// w (wl columns, repeated along the row), with silu(gate) applied before
// the norm or after it, or sigmoid(gate) after it (``sigm``).  L lanes a part: 8 to 64, or the workgroup.
// Up to KEEP vectors a lane stay in registers between the passes.
template <typename T, int L, bool GATE_FIRST, bool VEC>
__global__ __launch_bounds__(256) void gated_norm_kernel(
    T* __restrict__ out, int ld_out, const float* __restrict__ y,
    const T* __restrict__ gate, int ld, int g_off,
    const float* __restrict__ w, int wl, int parts, int groups, int S,
    bool sigm, float eps) {
  constexpr int N = VEC ? 8 : 1;
  constexpr int KEEP = L == 256 ? 4 : (VEC ? 1 : 8);
  __shared__ float red[4];
  const int part = blockIdx.x * (256 / L) + threadIdx.x / L;
  if (part >= parts) return;  // whole groups of L lanes
  const int lane = threadIdx.x % L;
  const int t = part / groups, g = part % groups;
  const int c0 = g * S;  // the part's first column
  const float* src = y + (size_t)t * groups * S + c0;
  const T* gt = gate + (size_t)t * ld + g_off + c0;
  auto fetch = [&](int i, float* f) {
    if (VEC) load8(src + i, f);
    else f[0] = src[i];
    if (GATE_FIRST) {
      float z[N];
      if (VEC) load8(gt + i, z);
      else z[0] = to_f(gt[i]);
#pragma unroll
      for (int j = 0; j < N; ++j) f[j] *= silu_f(z[j]);
    }
  };
  float keep[KEEP][N], ssq = 0.f;
#pragma unroll
  for (int n = 0; n < KEEP; ++n) {
    const int i = (lane + n * L) * N;
    if (i < S) {
      fetch(i, keep[n]);
#pragma unroll
      for (int j = 0; j < N; ++j) ssq += keep[n][j] * keep[n][j];
    }
  }
  for (int i = (lane + KEEP * L) * N; i < S; i += L * N) {
    float f[N];
    fetch(i, f);
#pragma unroll
    for (int j = 0; j < N; ++j) ssq += f[j] * f[j];
  }
  ssq = L == 8    ? row8_sum(ssq)
        : L == 16 ? row16_sum(ssq)
        : L == 32 ? half_wave_sum(ssq)
        : L == 64 ? wave_sum(ssq)
                  : block_sum_256(ssq, red);
  const float r = 1.f / sqrtf(ssq / S + eps);
  T* dst = out + (size_t)t * ld_out + c0;
  auto emit = [&](int i, float* f) {
    float wn[N];
    const int wi = (c0 + i) % wl;
    if (VEC) load8(w + wi, wn);
    else wn[0] = w[wi];
    float z[N];
    if (!GATE_FIRST) {
      if (VEC) load8(gt + i, z);
      else z[0] = to_f(gt[i]);
    }
#pragma unroll
    for (int j = 0; j < N; ++j) {
      f[j] *= r * wn[j];
      if (!GATE_FIRST) f[j] *= (sigm ? 1.f : z[j]) * sigmoid_f(z[j]);
    }
    if (VEC) store8(dst + i, f);
    else dst[i] = from_f<T>(f[0]);
  };
#pragma unroll
  for (int n = 0; n < KEEP; ++n) {
    const int i = (lane + n * L) * N;
    if (i < S) emit(i, keep[n]);
  }
  for (int i = (lane + KEEP * L) * N; i < S; i += L * N) {
    float f[N];
    fetch(i, f);
    emit(i, f);
  }
}

// out[r] = norm(x[index[r]]) in the storage type (index null: row r).
// ONE: w is a single number.  CENTRED: the row's mean is taken off first.
template <typename T, bool ONE, bool CENTRED>
__global__ __launch_bounds__(256) void norm_rows_kernel(
    T* __restrict__ out, const float* __restrict__ x,
    const int* __restrict__ index, const float* __restrict__ w,
    float w_offset, int width, float eps) {
  __shared__ float red[4], red2[4];
  const size_t src = (size_t)(index ? index[blockIdx.x] : blockIdx.x) * width;
  const size_t dst = (size_t)blockIdx.x * width;
  float ssq = 0.f, mean = 0.f;
  if (CENTRED) {
    float sum = 0.f;
    for (int i = threadIdx.x; i < width; i += 256) sum += x[src + i];
    mean = block_sum_256(sum, red2) / width;
  }
  if ((width & 7) == 0) {
    for (int i = threadIdx.x * 8; i < width; i += 2048) {
      float f[8];
      load8(x + src + i, f);
#pragma unroll
      for (int j = 0; j < 8; ++j) ssq += (f[j] - mean) * (f[j] - mean);
    }
    const float r = 1.f / sqrtf(block_sum_256(ssq, red) / width + eps);
    for (int i = threadIdx.x * 8; i < width; i += 2048) {
      float f[8], wr[8];
      load8(x + src + i, f);
      if (!ONE) load8(w + i, wr);
#pragma unroll
      for (int j = 0; j < 8; ++j)
        f[j] = (f[j] - mean) * r * (w_offset + (ONE ? w[0] : wr[j]));
      store8(out + dst + i, f);
    }
    return;
  }
  for (int i = threadIdx.x; i < width; i += 256)
    ssq += (x[src + i] - mean) * (x[src + i] - mean);
  const float r = 1.f / sqrtf(block_sum_256(ssq, red) / width + eps);
  for (int i = threadIdx.x; i < width; i += 256)
    out[dst + i] = from_f<T>((x[src + i] - mean) * r *
                             (w_offset + w[ONE ? 0 : i]));
}

// x += norm(y) w_post, h = norm(x) w_pre in the storage type: what lies
// between two sublayers whose outputs are normed as well as their inputs.
// y null: nothing is added; w_pre (and h) null: the sum alone.  CENTRED:
// layer norms, else RMS norms.  L threads a row, a wave or the workgroup;
// KEEP runs of N neighbours a thread stay in registers between the passes,
// the rest is read again.
template <typename T, int L, int N, int KEEP, bool CENTRED>
__global__ __launch_bounds__(256) void post_pre_norm_kernel(
    float* __restrict__ x, const T* __restrict__ y,
    const float* __restrict__ w_post, const float* __restrict__ w_pre,
    T* __restrict__ h, int n_tok, int width, float eps) {
  __shared__ float red[4][4];
  const int runs = width / N, tid = threadIdx.x % L;
  const int row = blockIdx.x * (256 / L) + threadIdx.x / L;
  if (row >= n_tok) return;  // whole waves
  const float inv = 1.f / width;
  float* xr = x + (size_t)row * width;
  const T* yr = y ? y + (size_t)row * width : nullptr;
  auto over_row = [](float s, float* red) {
    return L == WAVE ? wave_sum(s) : block_sum_256(s, red);
  };
  auto load = [](const auto* p, float* f) {
    if constexpr (N == 8) load8(p, f);
    else f[0] = to_f(p[0]);
  };
  auto store = [](auto* p, const float* f) {
    using S = std::remove_reference_t<decltype(*p)>;
    if constexpr (N == 8) store8(p, f);
    else p[0] = from_f<S>(f[0]);
  };
  float keep[KEEP][N], mean = 0.f;
  // sums over the row of ``src``, of which the first runs are kept
  auto total = [&](const auto* src, float* red) {
    float s = 0.f;
#pragma unroll
    for (int k = 0; k < KEEP; ++k)
      if (tid + k * L < runs)
#pragma unroll
        for (int j = 0; j < N; ++j) s += keep[k][j];
    for (int i = tid + KEEP * L; i < runs; i += L) {
      float f[N];
      load(src + (size_t)i * N, f);
#pragma unroll
      for (int j = 0; j < N; ++j) s += f[j];
    }
    return over_row(s, red);
  };
  auto squares = [&](const auto* src, float* red) {
    float s = 0.f;
#pragma unroll
    for (int k = 0; k < KEEP; ++k)
      if (tid + k * L < runs)
#pragma unroll
        for (int j = 0; j < N; ++j)
          s += (keep[k][j] - mean) * (keep[k][j] - mean);
    for (int i = tid + KEEP * L; i < runs; i += L) {
      float f[N];
      load(src + (size_t)i * N, f);
#pragma unroll
      for (int j = 0; j < N; ++j) s += (f[j] - mean) * (f[j] - mean);
    }
    return over_row(s, red);
  };
  if (y) {
    // the stream's loads fly behind the norm of y
    float xk[KEEP][N];
#pragma unroll
    for (int k = 0; k < KEEP; ++k)
      if (tid + k * L < runs) load(yr + (size_t)(tid + k * L) * N, keep[k]);
#pragma unroll
    for (int k = 0; k < KEEP; ++k)
      if (tid + k * L < runs) load(xr + (size_t)(tid + k * L) * N, xk[k]);
    if (CENTRED) mean = total(yr, red[0]) * inv;
    const float r = 1.f / sqrtf(squares(yr, red[1]) * inv + eps);
    auto add = [&](int i, const float* f, float* out) {
      float w[N];
      load(w_post + (size_t)i * N, w);
#pragma unroll
      for (int j = 0; j < N; ++j) out[j] += (f[j] - mean) * r * w[j];
      store(xr + (size_t)i * N, out);
    };
#pragma unroll
    for (int k = 0; k < KEEP; ++k)
      if (tid + k * L < runs) {
        add(tid + k * L, keep[k], xk[k]);
#pragma unroll
        for (int j = 0; j < N; ++j) keep[k][j] = xk[k][j];
      }
    for (int i = tid + KEEP * L; i < runs; i += L) {
      float f[N], v[N];
      load(yr + (size_t)i * N, f);
      load(xr + (size_t)i * N, v);
      add(i, f, v);
    }
  } else {
#pragma unroll
    for (int k = 0; k < KEEP; ++k)
      if (tid + k * L < runs) load(xr + (size_t)(tid + k * L) * N, keep[k]);
  }
  if (!w_pre) return;
  // beyond the kept runs a thread reads back only what it wrote itself
  mean = 0.f;
  if (CENTRED) mean = total(xr, red[2]) * inv;
  const float r = 1.f / sqrtf(squares(xr, red[3]) * inv + eps);
  T* hr = h + (size_t)row * width;
  auto emit = [&](int i, float* f) {
    float w[N];
    load(w_pre + (size_t)i * N, w);
#pragma unroll
    for (int j = 0; j < N; ++j) f[j] = (f[j] - mean) * r * w[j];
    store(hr + (size_t)i * N, f);
  };
#pragma unroll
  for (int k = 0; k < KEEP; ++k)
    if (tid + k * L < runs) emit(tid + k * L, keep[k]);
  for (int i = tid + KEEP * L; i < runs; i += L) {
    float f[N];
    load(xr + (size_t)i * N, f);
    emit(i, f);
  }
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

// out = g sigmoid(sharpness g) (u + 1) with g = min(gate, limit) and
// u = clamp(up, -limit, limit); gate and up lie u_off columns apart.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void clamped_swiglu_kernel(
    T* __restrict__ out, int ld_out, const T* __restrict__ gu, int ld,
    int u_off, int n_tok, int ff, float limit, float sharpness) {
  constexpr int N = VEC ? 8 : 1;
  const int per_row = ff / N;
  const long long total = (long long)n_tok * per_row;
  const long long step = (long long)gridDim.x * 256;
  for (long long id = (long long)blockIdx.x * 256 + threadIdx.x; id < total;
       id += step) {
    const int t = (int)(id / per_row);
    const int i = (int)(id - (long long)t * per_row) * N;
    const T* src = gu + (size_t)t * ld + i;
    float g[N], u[N];
    if (VEC) {
      load8(src, g);
      load8(src + u_off, u);
    } else {
      g[0] = to_f(src[0]);
      u[0] = to_f(src[u_off]);
    }
#pragma unroll
    for (int j = 0; j < N; ++j) {
      g[j] = fminf(g[j], limit);
      u[j] = fminf(fmaxf(u[j], -limit), limit);
      const float e = sizeof(T) == 2 ? __expf(-sharpness * g[j])
                                     : expf(-sharpness * g[j]);
      g[j] = g[j] / (1.f + e) * (u[j] + 1.f);
    }
    T* dst = out + (size_t)t * ld_out + i;
    if (VEC) store8(dst, g);
    else dst[0] = from_f<T>(g[0]);
  }
}

// out = max(u, 0)^2
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void squared_relu_kernel(
    T* __restrict__ out, int ld_out, const T* __restrict__ u, int ld,
    int n_tok, int ff) {
  constexpr int N = VEC ? 8 : 1;
  const int per_row = ff / N;
  const long long total = (long long)n_tok * per_row;
  const long long step = (long long)gridDim.x * 256;
  for (long long id = (long long)blockIdx.x * 256 + threadIdx.x; id < total;
       id += step) {
    const int t = (int)(id / per_row);
    const int i = (int)(id - (long long)t * per_row) * N;
    const T* src = u + (size_t)t * ld + i;
    float f[N];
    if (VEC) load8(src, f);
    else f[0] = to_f(src[0]);
#pragma unroll
    for (int j = 0; j < N; ++j) {
      f[j] = fmaxf(f[j], 0.f);
      f[j] *= f[j];
    }
    T* dst = out + (size_t)t * ld_out + i;
    if (VEC) store8(dst, f);
    else dst[0] = from_f<T>(f[0]);
  }
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
                 int one, float w_offset, int centred, int n_rows, int width,
                 float eps, int dtype, void* stream) {
  if (n_rows <= 0) return 0;
#define GO(ONE, CENTRED)                                                     \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                        \
      (norm_rows_kernel<T, ONE, CENTRED>), dim3(n_rows), dim3(256), 0,       \
      (hipStream_t)stream, (T*)out, (const float*)x, (const int*)index,      \
      (const float*)w, w_offset, width, eps))
  if (one && centred) GO(true, true);
  else if (one) GO(true, false);
  else if (centred) GO(false, true);
  else GO(false, false);
#undef GO
  HY_CHECK();
  return 0;
}

int hy_post_pre_norm(void* x, const void* y, const void* w_post,
                     const void* w_pre, void* h, int centred, int n_tok,
                     int width, float eps, int dtype, void* stream) {
  if ((y && !w_post) || (w_pre && !h) || width <= 0) return -2;
  if (n_tok <= 0) return 0;
#define GO(L, N, KEEP, CENTRED)                                              \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                        \
      (post_pre_norm_kernel<T, L, N, KEEP, CENTRED>),                        \
      dim3((n_tok + 256 / L - 1) / (256 / L)), dim3(256), 0,                 \
      (hipStream_t)stream, (float*)x, (const T*)y, (const float*)w_post,     \
      (const float*)w_pre, (T*)h, n_tok, width, eps))
#define PICK(L, N, KEEP)                 \
  do {                                   \
    if (centred) GO(L, N, KEEP, true);   \
    else GO(L, N, KEEP, false);          \
  } while (0)
  // a wave a row where there are rows enough for all of them
  const bool many = n_tok >= 2048;
  if (width % 8) PICK(256, 1, 4);
  else if (many && width <= 512) PICK(64, 8, 1);
  else if (many && width <= 1024) PICK(64, 8, 2);
  else if (width <= 2048) PICK(256, 8, 1);
  else if (width <= 4096) PICK(256, 8, 2);
  else PICK(256, 8, 4);
#undef PICK
#undef GO
  HY_CHECK();
  return 0;
}

int hy_add_norms(void* x, const void* y, const void* z, const void* zw,
                 int top, float mult, const void* w1, const void* w2,
                 int one, void* h1, void* h2, int n_tok, int width, float eps,
                 int dtype, void* stream) {
  if ((w1 && !h1) || (w2 && (!h2 || !w1))) return -2;
  if (z && (!y || !zw || top < 1)) return -2;
  if (n_tok <= 0) return 0;
#define GO(ROUTED, ONE)                                                      \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                        \
      (add_norms_kernel<T, ROUTED, ONE>), dim3(n_tok), dim3(256), 0,         \
      (hipStream_t)stream, (float*)x, (const T*)y, (const T*)z,              \
      (const float*)zw, top, mult, (const float*)w1, (const float*)w2,       \
      (T*)h1, (T*)h2, width, eps))
  if (z && one) GO(true, true);
  else if (z) GO(true, false);
  else if (one) GO(false, true);
  else GO(false, false);
#undef GO
  HY_CHECK();
  return 0;
}

int hy_gated_norm(void* out, int ld_out, const void* y, const void* gate,
                  int ld, int g_off, const void* w, int wl, int n_tok,
                  int groups, int S, int gate_first, int sigm, float eps,
                  int dtype, void* stream) {
  if (sigm && gate_first) return -2;
  if (groups <= 0 || S <= 0 || wl <= 0 || (groups * S) % wl) return -2;
  if (n_tok <= 0) return 0;
  if ((long long)n_tok * groups >= (1ll << 31)) return -2;
  const int parts = n_tok * groups;
  const bool vec = S % 8 == 0 && wl % 8 == 0 && ld % 8 == 0 &&
                   ld_out % 8 == 0 && g_off % 8 == 0;
#define GO(L, FIRST, VEC)                                                   \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                       \
      (gated_norm_kernel<T, L, FIRST, VEC>),                                \
      dim3((parts + 256 / L - 1) / (256 / L)), dim3(256), 0,                \
      (hipStream_t)stream, (T*)out, ld_out, (const float*)y,                \
      (const T*)gate, ld, g_off, (const float*)w, wl, parts, groups, S,     \
      sigm != 0, eps))
#define PICK(L)                                \
  do {                                         \
    if (gate_first && vec) GO(L, true, true);  \
    else if (gate_first) GO(L, true, false);   \
    else if (vec) GO(L, false, true);          \
    else GO(L, false, false);                  \
  } while (0)
  if (S <= 64) PICK(8);
  else if (S <= 128) PICK(16);
  else if (S <= 256) PICK(32);
  else if (S <= 512) PICK(64);
  else PICK(256);
#undef PICK
#undef GO
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

int hy_clamped_swiglu(void* out, int ld_out, const void* gu, int ld,
                      int u_off, int n_tok, int ff, float limit,
                      float sharpness, int dtype, void* stream) {
  if (n_tok <= 0 || ff <= 0) return 0;
  const bool vec =
      ff % 8 == 0 && ld % 8 == 0 && ld_out % 8 == 0 && u_off % 8 == 0 &&
      ((uintptr_t)out & (dtype == 0 ? 15 : 31)) == 0;
  const int grid = grid_for((long long)n_tok * ff / (vec ? 8 : 1));
#define GO(VEC)                                                            \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                      \
      (clamped_swiglu_kernel<T, VEC>), dim3(grid), dim3(256), 0,           \
      (hipStream_t)stream, (T*)out, ld_out, (const T*)gu, ld, u_off, n_tok, \
      ff, limit, sharpness))
  if (vec) GO(true);
  else GO(false);
#undef GO
  HY_CHECK();
  return 0;
}

int hy_squared_relu(void* out, int ld_out, const void* u, int ld, int n_tok,
                    int ff, int dtype, void* stream) {
  if (n_tok <= 0 || ff <= 0) return 0;
  const uintptr_t mask = dtype == 0 ? 15 : 31;
  const bool vec = ff % 8 == 0 && ld % 8 == 0 && ld_out % 8 == 0 &&
                   (((uintptr_t)out | (uintptr_t)u) & mask) == 0;
  const int grid = grid_for((long long)n_tok * ff / (vec ? 8 : 1));
#define GO(VEC)                                                              \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                        \
      (squared_relu_kernel<T, VEC>), dim3(grid), dim3(256), 0,               \
      (hipStream_t)stream, (T*)out, ld_out, (const T*)u, ld, n_tok, ff))
  if (vec) GO(true);
  else GO(false);
#undef GO
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
