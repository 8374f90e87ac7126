// Routing of tokens to experts: logits W h in 32-bit, softmax over all
// experts, the ``top`` largest scores among the ``keep`` groups of
// neighbours with the largest best score, divided by their sum.
//
//   index [T][top] experts, weight [T][top]; with ``counts`` (zeroed by
//   the caller) also the experts' lists (experts.h)
//
//  * route_mfma_kernel  bf16: 16 MT tokens a workgroup, the depth split
//    over its waves
//  * route_rows_kernel  any size and either type, a workgroup a token
#include "experts.h"
#include "mfma.h"

// One wave: choose for one token from its E logits (LDS, replaced by the
// scores); ``best`` holds ``groups`` floats, ``open`` as many flags.
__device__ __forceinline__ void choose_experts(
    float* s, float* best, int* open, int E, int top, int groups, int keep,
    float scale, int* __restrict__ index, float* __restrict__ weight) {
  const int lane = threadIdx.x & (WAVE - 1);
  float m = -INFINITY, sum = 0.f;
  for (int e = lane; e < E; e += WAVE) m = fmaxf(m, s[e]);
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) m = fmaxf(m, __shfl_xor(m, o, WAVE));
  for (int e = lane; e < E; e += WAVE) {
    const float x = expf(s[e] - m);
    s[e] = x >= 0.f ? x : 0.f;  // scores stay ordered whatever the logits
    sum += s[e];
  }
  sum = wave_sum(sum);
  const float inv = sum > 0.f ? 1.f / sum : 0.f;
  for (int e = lane; e < E; e += WAVE) s[e] *= inv;
  __builtin_amdgcn_wave_barrier();
  const int size = E / groups;
  for (int g = lane; g < groups; g += WAVE) {
    float b = s[g * size];
    for (int i = 1; i < size; ++i) b = fmaxf(b, s[g * size + i]);
    best[g] = b;
  }
  __builtin_amdgcn_wave_barrier();
  for (int g = lane; g < groups; g += WAVE) {
    int rank = 0;  // groups that come before this one
    for (int i = 0; i < groups; ++i)
      rank += best[i] > best[g] || (best[i] == best[g] && i < g);
    open[g] = rank < keep;
  }
  __builtin_amdgcn_wave_barrier();
  float taken = 0.f;
  for (int e = lane; e < E; e += WAVE) {
    if (!open[e / size]) continue;
    const float x = s[e];
    int rank = 0;
    for (int g = 0; g < groups; ++g) {
      if (!open[g]) continue;
      for (int i = g * size; i < (g + 1) * size; ++i)
        rank += s[i] > x || (s[i] == x && i < e);
    }
    if (rank < top) {
      index[rank] = e;
      weight[rank] = x;
      taken += x;
    }
  }
  const float f = scale / (wave_sum(taken) + 1e-20f);
  __builtin_amdgcn_wave_barrier();
  for (int k = lane; k < top; k += WAVE) weight[k] *= f;
}

// LDS of the choice, per wave: groups floats and groups ints
#define CHOICE_BYTES(groups) ((groups) * 8)

template <typename T>
__global__ __launch_bounds__(256) void route_rows_kernel(
    int* __restrict__ index, float* __restrict__ weight,
    int* __restrict__ counts, int* __restrict__ pairs,
    const T* __restrict__ h, const T* __restrict__ w, int width, int E,
    int top, int groups, int keep, float scale, int n_tok) {
  extern __shared__ float lds[];
  float* s = lds;                          // E logits
  float* best = s + E;                     // groups
  int* open = (int*)(best + groups);       // groups
  int* idx = open + groups;                // top
  float* wgt = (float*)(idx + top);        // top
  const int t = blockIdx.x, wave = threadIdx.x / WAVE;
  const int lane = threadIdx.x & (WAVE - 1);
  const T* x = h + (size_t)t * width;
  for (int e = wave; e < E; e += 4) {
    const T* r = w + (size_t)e * width;
    float a = 0.f;
    for (int i = lane; i < width; i += WAVE) a += to_f(x[i]) * to_f(r[i]);
    a = wave_sum(a);
    if (lane == 0) s[e] = a;
  }
  __syncthreads();
  if (wave != 0) return;
  choose_experts(s, best, open, E, top, groups, keep, scale, idx, wgt);
  __builtin_amdgcn_wave_barrier();
  for (int k = lane; k < top; k += WAVE) {
    index[(size_t)t * top + k] = idx[k];
    weight[(size_t)t * top + k] = wgt[k];
    if (counts)
      pairs[(size_t)idx[k] * n_tok + atomicAdd(&counts[idx[k]], 1)] =
          t * top + k;
  }
}

// LDS: red [NW][16 MT][16 NT + 4] floats, logits [16 MT][E], then per wave
// the choice's, then idx and wgt [16 MT][top], hist and base [E]
template <int MT, int NT, int NW>
__global__ __launch_bounds__(NW * 64) void route_mfma_kernel(
    int* __restrict__ index, float* __restrict__ weight,
    int* __restrict__ counts, int* __restrict__ pairs,
    const bf16_t* __restrict__ h, const bf16_t* __restrict__ w, int width,
    int E, int top, int groups, int keep, float scale, int n_tok) {
  constexpr int TM = 16 * MT, RP = 16 * NT + 4;
  extern __shared__ float lds[];
  float* red = lds;
  float* logits = red + NW * TM * RP;
  float* choice = logits + TM * E;
  int* idx = (int*)(choice + NW * 2 * groups);
  float* wgt = (float*)(idx + TM * top);
  int* hist = (int*)(wgt + TM * top);
  int* base = hist + E;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & 63;
  const int n = lane & 15, g = lane >> 4;
  const int t0 = blockIdx.x * TM;
  const bf16_t* hp[MT];
#pragma unroll
  for (int a = 0; a < MT; ++a) {
    const int t = t0 + a * 16 + n;
    hp[a] = h + (size_t)(t < n_tok ? t : n_tok - 1) * width;
  }
  for (int e = tid; e < E; e += NW * 64) hist[e] = 0;
  for (int e0 = 0; e0 < E; e0 += 16 * NT) {
    const bf16_t* wp[NT];
#pragma unroll
    for (int b = 0; b < NT; ++b) {
      const int e = e0 + b * 16 + n;
      wp[b] = w + (size_t)(e < E ? e : E - 1) * width;
    }
    f32x4 acc[MT][NT];
#pragma unroll
    for (int a = 0; a < MT; ++a)
#pragma unroll
      for (int b = 0; b < NT; ++b) acc[a][b] = f32x4{0.f, 0.f, 0.f, 0.f};
    // 64 numbers of the depth at a time; past its end tokens count as zero
#pragma unroll 2
    for (int k0 = wave * 64; k0 < width; k0 += NW * 64) {
      u32x4 hf[2][MT], wf[2][NT];
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        const int k = k0 + s * 32 + g * 8;
        const bool in = k < width;
        const int kk = in ? k : 0;
#pragma unroll
        for (int a = 0; a < MT; ++a) {
          hf[s][a] = *reinterpret_cast<const u32x4*>(hp[a] + kk);
          if (!in) hf[s][a] = u32x4{0, 0, 0, 0};
        }
#pragma unroll
        for (int b = 0; b < NT; ++b)
          wf[s][b] = *reinterpret_cast<const u32x4*>(wp[b] + kk);
      }
#pragma unroll
      for (int s = 0; s < 2; ++s)
#pragma unroll
        for (int a = 0; a < MT; ++a)
#pragma unroll
          for (int b = 0; b < NT; ++b)
            acc[a][b] = mfma(wf[s][b], hf[s][a], acc[a][b]);
    }
    // a lane holds experts 4g..4g+3 of token n
#pragma unroll
    for (int a = 0; a < MT; ++a)
#pragma unroll
      for (int b = 0; b < NT; ++b)
        *reinterpret_cast<f32x4*>(
            &red[(wave * TM + a * 16 + n) * RP + b * 16 + g * 4]) = acc[a][b];
    __syncthreads();
    for (int i = tid; i < TM * 16 * NT; i += NW * 64) {
      const int t = i / (16 * NT), e = i % (16 * NT);
      float x = 0.f;
#pragma unroll
      for (int v = 0; v < NW; ++v) x += red[(v * TM + t) * RP + e];
      if (e0 + e < E) logits[t * E + e0 + e] = x;
    }
    __syncthreads();
  }
  float* best = choice + wave * 2 * groups;
  for (int i = wave; i < TM; i += NW) {
    if (t0 + i >= n_tok) break;
    choose_experts(logits + i * E, best, (int*)(best + groups), E, top,
                   groups, keep, scale, idx + i * top, wgt + i * top);
    __builtin_amdgcn_wave_barrier();
  }
  __syncthreads();
  const int n_pairs = (n_tok - t0 < TM ? n_tok - t0 : TM) * top;
  for (int i = tid; i < n_pairs; i += NW * 64) {
    index[(size_t)t0 * top + i] = idx[i];
    weight[(size_t)t0 * top + i] = wgt[i];
  }
  if (!counts) return;
  // places in the experts' lists: one reservation an expert
  int* rank = (int*)red;
  for (int i = tid; i < n_pairs; i += NW * 64)
    rank[i] = atomicAdd(&hist[idx[i]], 1);
  __syncthreads();
  for (int e = tid; e < E; e += NW * 64)
    if (hist[e]) base[e] = atomicAdd(&counts[e], hist[e]);
  __syncthreads();
  for (int i = tid; i < n_pairs; i += NW * 64)
    pairs[(size_t)idx[i] * n_tok + base[idx[i]] + rank[i]] = t0 * top + i;
}

extern "C" {

int hy_route(void* index, void* weight, void* counts, void* pairs,
             const void* h, const void* w, int width, int E, int top,
             int groups, int keep, float scale, int n_tok, int dtype,
             void* stream) {
  if (width <= 0 || E <= 0 || E > 1024 || groups <= 0 || E % groups ||
      keep < 1 || keep > groups || top < 1 || top > keep * (E / groups) ||
      (counts && !pairs))
    return -2;
  if (n_tok <= 0) return 0;
  if ((long long)n_tok * top >= (1ll << 31)) return -2;
#define ARGS                                                             \
  (hipStream_t)stream, (int*)index, (float*)weight, (int*)counts,        \
      (int*)pairs, (const T*)h, (const T*)w, width, E, top, groups, keep, \
      scale, n_tok
  if (dtype == 0 && width % 8 == 0 && E <= 256 && groups <= 64 &&
      top <= 32) {
    using T = bf16_t;
#define GO(MT, NT, NW)                                                      \
  hipLaunchKernelGGL(                                                       \
      (route_mfma_kernel<MT, NT, NW>), dim3((n_tok + 16 * MT - 1) /         \
                                            (16 * MT)),                     \
      dim3(NW * 64),                                                        \
      4 * (NW * 16 * MT * (16 * NT + 4) + 16 * MT * E + NW * 2 * groups +   \
           2 * 16 * MT * top + 2 * E),                                      \
      ARGS)
    if (n_tok <= 2048) {
      if (E <= 16) GO(1, 1, 8);
      else if (E <= 32) GO(1, 2, 8);
      else GO(1, 4, 8);
    } else {
      if (E <= 16) GO(2, 1, 4);
      else if (E <= 32) GO(2, 2, 4);
      else GO(1, 4, 4);
    }
#undef GO
  } else {
    HY_DTYPE(dtype, hipLaunchKernelGGL(
        route_rows_kernel<T>, dim3(n_tok), dim3(256),
        4 * (E + 2 * groups + 2 * top), ARGS));
  }
#undef ARGS
  HY_CHECK();
  return 0;
}

}  // extern "C"
