// Routing kernels (router.h):
//  * route_kernel       bf16, 16 tokens a workgroup on the matrix cores
//  * route_rows_kernel  any size and either type, a workgroup a token
#include "router.h"

template <int NT>
__global__ __launch_bounds__(256) void route_kernel(Routing a) {
  extern __shared__ float lds[];
  route_block<NT>(a, blockIdx.x, lds);
}

template <typename T>
__global__ __launch_bounds__(256) void route_rows_kernel(Routing a) {
  extern __shared__ float lds[];
  const int E = a.E, top = a.top;
  float* s = lds;                          // E logits
  float* best = s + E;                     // groups
  int* open = (int*)(best + a.groups);     // groups
  int* idx = open + a.groups;              // top
  float* wgt = (float*)(idx + top);        // top
  const int t = blockIdx.x, wave = threadIdx.x / WAVE;
  const int lane = threadIdx.x & (WAVE - 1);
  const T* x = (const T*)a.h + (size_t)t * a.width;
  for (int e = wave; e < E; e += 4) {
    const T* r = (const T*)a.w + (size_t)e * a.width;
    float acc = 0.f;
    for (int i = lane; i < a.width; i += WAVE) acc += to_f(x[i]) * to_f(r[i]);
    acc = wave_sum(acc);
    if (lane == 0) s[e] = acc;
  }
  __syncthreads();
  if (wave != 0) return;
  choose_experts(s, best, open, E, top, a.groups, a.keep, a.scale, idx, wgt);
  __builtin_amdgcn_wave_barrier();
  for (int k = lane; k < top; k += WAVE) {
    a.index[(size_t)t * top + k] = idx[k];
    a.weight[(size_t)t * top + k] = wgt[k];
    if (a.counts)
      a.pairs[(size_t)idx[k] * a.n_tok + atomicAdd(&a.counts[idx[k]], 1)] =
          t * top + k;
  }
}

extern "C" int hy_route(void* index, void* weight, void* counts, void* pairs,
                        const void* h, const void* w, int width, int E,
                        int top, int groups, int keep, float scale, int n_tok,
                        int dtype, void* stream) {
  const Routing a{(int*)index, (float*)weight, (int*)counts, (int*)pairs, h,
                  w, width, E, top, groups, keep, scale, n_tok};
  if (!routing_ok(a)) return -2;
  if (n_tok <= 0) return 0;
  const hipStream_t st = (hipStream_t)stream;
  if (route_block_ok(a, dtype)) {
    const dim3 grid((n_tok + 15) / 16), block(256);
#define GO(NT)                                                            \
  hipLaunchKernelGGL(route_kernel<NT>, grid, block,                       \
                     4 * route_floats<NT>(E, top, groups), st, a)
    if (E <= 16) GO(1);
    else if (E <= 32) GO(2);
    else GO(4);
#undef GO
  } else {
    HY_DTYPE(dtype, hipLaunchKernelGGL(
        route_rows_kernel<T>, dim3(n_tok), dim3(256),
        4 * (E + 2 * groups + 2 * top), st, a));
  }
  HY_CHECK();
  return 0;
}
