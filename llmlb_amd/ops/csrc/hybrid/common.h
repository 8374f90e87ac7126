// Shared helpers of the hybrid-model kernels (gfx950, wave64).
//
// Every kernel is a template over the storage type of activations and
// weights: bf16 (raw 16-bit) or float.  Arithmetic is float throughout.
#pragma once
#include <hip/hip_runtime.h>
#include <math.h>
#include <stdint.h>
#include <type_traits>

#define WAVE 64
#define PAGE 16  // tokens per cache page

struct bf16_t {
  unsigned short u;
};

__device__ __forceinline__ float to_f(float x) { return x; }
__device__ __forceinline__ float to_f(bf16_t x) {
  return __uint_as_float((unsigned)x.u << 16);
}

template <typename T>
__device__ __forceinline__ T from_f(float f);
template <>
__device__ __forceinline__ float from_f<float>(float f) { return f; }
// round to nearest even
template <>
__device__ __forceinline__ bf16_t from_f<bf16_t>(float f) {
  unsigned x = __float_as_uint(f);
  bf16_t r;
  r.u = (unsigned short)((x + 0x7FFFu + ((x >> 16) & 1u)) >> 16);
  return r;
}

// 8 consecutive elements; the address is 16-byte aligned
__device__ __forceinline__ void load8(const bf16_t* p, float* f) {
  const uint4 v = *reinterpret_cast<const uint4*>(p);
  f[0] = __uint_as_float(v.x << 16); f[1] = __uint_as_float(v.x & 0xffff0000u);
  f[2] = __uint_as_float(v.y << 16); f[3] = __uint_as_float(v.y & 0xffff0000u);
  f[4] = __uint_as_float(v.z << 16); f[5] = __uint_as_float(v.z & 0xffff0000u);
  f[6] = __uint_as_float(v.w << 16); f[7] = __uint_as_float(v.w & 0xffff0000u);
}
__device__ __forceinline__ void load8(const float* p, float* f) {
  const float4 a = reinterpret_cast<const float4*>(p)[0];
  const float4 b = reinterpret_cast<const float4*>(p)[1];
  f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w;
  f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
}
__device__ __forceinline__ unsigned pack2(float lo, float hi) {
  return (unsigned)from_f<bf16_t>(lo).u |
         ((unsigned)from_f<bf16_t>(hi).u << 16);
}
__device__ __forceinline__ void store8(bf16_t* p, const float* f) {
  uint4 v;
  v.x = pack2(f[0], f[1]); v.y = pack2(f[2], f[3]);
  v.z = pack2(f[4], f[5]); v.w = pack2(f[6], f[7]);
  *reinterpret_cast<uint4*>(p) = v;
}
__device__ __forceinline__ void store8(float* p, const float* f) {
  reinterpret_cast<float4*>(p)[0] = make_float4(f[0], f[1], f[2], f[3]);
  reinterpret_cast<float4*>(p)[1] = make_float4(f[4], f[5], f[6], f[7]);
}

// 4 consecutive elements; the address is aligned to all four
__device__ __forceinline__ void load4(const bf16_t* p, float* f) {
  const uint2 v = *reinterpret_cast<const uint2*>(p);
  f[0] = __uint_as_float(v.x << 16); f[1] = __uint_as_float(v.x & 0xffff0000u);
  f[2] = __uint_as_float(v.y << 16); f[3] = __uint_as_float(v.y & 0xffff0000u);
}
__device__ __forceinline__ void load4(const float* p, float* f) {
  const float4 v = *reinterpret_cast<const float4*>(p);
  f[0] = v.x; f[1] = v.y; f[2] = v.z; f[3] = v.w;
}
__device__ __forceinline__ void store4(bf16_t* p, const float* f) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack2(f[0], f[1]),
                                            pack2(f[2], f[3]));
}
__device__ __forceinline__ void store4(float* p, const float* f) {
  *reinterpret_cast<float4*>(p) = make_float4(f[0], f[1], f[2], f[3]);
}

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, WAVE);
  return v;
}

// sum over a 256-thread workgroup; ``red`` holds 4 floats
__device__ __forceinline__ float block_sum_256(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & (WAVE - 1)) == 0) red[threadIdx.x / WAVE] = v;
  __syncthreads();
  return red[0] + red[1] + red[2] + red[3];
}

// sum over each group of 16 consecutive lanes, without LDS traffic
template <int CTRL>
__device__ __forceinline__ float dpp_add(float v) {
  return v + __int_as_float(__builtin_amdgcn_update_dpp(
                 0, __float_as_int(v), CTRL, 0xf, 0xf, true));
}
__device__ __forceinline__ float row16_sum(float v) {
  v = dpp_add<0xB1>(v);   // quad_perm [1,0,3,2]
  v = dpp_add<0x4E>(v);   // quad_perm [2,3,0,1]
  v = dpp_add<0x141>(v);  // row_half_mirror
  v = dpp_add<0x140>(v);  // row_mirror
  return v;
}

__device__ __forceinline__ float row8_sum(float v) {  // of 8 lanes
  v = dpp_add<0xB1>(v);
  v = dpp_add<0x4E>(v);
  return dpp_add<0x141>(v);
}
__device__ __forceinline__ float half_wave_sum(float v) {  // of 32 lanes
  v = row16_sum(v);
  return v + __shfl_xor(v, 16, WAVE);
}
// Four sums over 16 lanes at once: lane l gets the one of v[l % 4].
__device__ __forceinline__ float row16_sum4(const float* v) {
  const bool odd = threadIdx.x & 1, high = threadIdx.x & 2;
  float a = odd ? v[1] : v[0], b = odd ? v[3] : v[2];
  const float a2 = odd ? v[0] : v[1], b2 = odd ? v[2] : v[3];
  auto from = [](float x, auto ctrl) {
    return __int_as_float(__builtin_amdgcn_update_dpp(
        0, __float_as_int(x), decltype(ctrl)::value, 0xf, 0xf, true));
  };
  a += from(a2, std::integral_constant<int, 0xB1>());  // lane ^ 1
  b += from(b2, std::integral_constant<int, 0xB1>());
  float c = high ? b : a;
  const float c2 = high ? a : b;
  c += from(c2, std::integral_constant<int, 0x4E>());  // lane ^ 2
  c = dpp_add<0x124>(c);                               // row_ror:4
  return dpp_add<0x128>(c);                            // row_ror:8
}

__device__ __forceinline__ float sigmoid_f(float x) {
  return 1.f / (1.f + expf(-x));
}
__device__ __forceinline__ float silu_f(float x) { return x * sigmoid_f(x); }
__device__ __forceinline__ float softplus_f(float x) {
  return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x)));
}

// flat token slot of position ``pos`` of the sequence in table row ``row``
__device__ __forceinline__ size_t page_slot(const int* bt, int max_blocks,
                                            int row, int pos) {
  return (size_t)bt[(size_t)row * max_blocks + pos / PAGE] * PAGE +
         pos % PAGE;
}

// Which keys the query at position i sees: the last ``size`` ones, or those
// of its own chunk of ``size`` positions.
struct Mask {
  int size;
  bool chunk;
  // how far back the first of them lies (it may be before position 0)
  __device__ __forceinline__ int span(int i) const {
    return chunk ? i % size : size - 1;
  }
  __device__ __forceinline__ int first(int i) const {
    const int j = i - span(i);
    return j > 0 ? j : 0;
  }
};

#define HY_CHECK()                                  \
  do {                                              \
    if (hipGetLastError() != hipSuccess) return -1; \
  } while (0)

// dispatch on the storage type: 0 = bf16, 1 = float
#define HY_DTYPE(dtype, ...)                  \
  do {                                        \
    if ((dtype) == 0) {                       \
      using T = bf16_t;                       \
      __VA_ARGS__;                            \
    } else {                                  \
      using T = float;                        \
      __VA_ARGS__;                            \
    }                                         \
  } while (0)
