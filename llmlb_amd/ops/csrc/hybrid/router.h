// Routing of tokens to experts: logits W h in 32-bit, softmax over all
// experts, the ``top`` largest scores among the ``keep`` groups of
// neighbours with the largest best score, divided by their sum.
#pragma once
#include "experts.h"
#include "mfma.h"

struct Routing {
  int* index;     // [T][top] experts
  float* weight;  // [T][top]
  int* counts;    // null, or zeroed by the caller: lists (experts.h) too
  int* pairs;
  const void* h;
  const void* w;
  int width, E, top, groups, keep;
  float scale;
  int n_tok;
};

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

// 64 / L tokens a wave, an expert a lane (E <= L): the same choice in
// registers.  ``s``: this lane's logit; idx, wgt: the token's in LDS.
template <int L>
__device__ __forceinline__ void choose_experts_lane(float s, int E, int top,
                                                    int groups, int keep,
                                                    float scale, int* idx,
                                                    float* wgt) {
  const int e = threadIdx.x % L;
  const bool real = e < E;
  float m = real ? s : -INFINITY;
#pragma unroll
  for (int o = L / 2; o > 0; o >>= 1) m = fmaxf(m, __shfl_xor(m, o, L));
  float x = expf(s - m);
  x = real && x >= 0.f ? x : 0.f;
  float sum = x;
#pragma unroll
  for (int o = L / 2; o > 0; o >>= 1) sum += __shfl_xor(sum, o, L);
  x *= sum > 0.f ? 1.f / sum : 0.f;
  const int size = E / groups, g = real ? e / size : 0;
  float best = 0.f;
  for (int i = 0; i < size; ++i)
    best = fmaxf(best, __shfl(x, g * size + i, L));
  int rank = 0;  // groups that come before this one
  for (int i = 0; i < groups; ++i) {
    const float b = __shfl(best, i * size, L);
    rank += b > best || (b == best && i < g);
  }
  const float y = real && rank < keep ? x : -1.f;
  rank = 0;
#pragma unroll 8
  for (int i = 0; i < L; ++i) {
    const float b = __shfl(y, i, L);
    rank += b > y || (b == y && i < e);
  }
  const bool mine = y >= 0.f && rank < top;
  sum = mine ? x : 0.f;
#pragma unroll
  for (int o = L / 2; o > 0; o >>= 1) sum += __shfl_xor(sum, o, L);
  if (mine) {
    idx[rank] = e;
    wgt[rank] = x * (scale / (sum + 1e-20f));
  }
}

// A workgroup of four waves routes 16 tokens (bf16), the depth split over
// the waves, 16 NT experts at a time.  LDS, in floats:
//   red [4][16][16 NT + 4], logits [16][E], the choice's [4][2 groups],
//   idx and wgt [16][top], hist and base [E]
template <int NT>
__host__ __device__ constexpr int route_floats(int E, int top, int groups) {
  return 4 * 16 * (16 * NT + 4) + 16 * E + 8 * groups + 32 * top + 2 * E;
}
template <int NT>
__device__ __forceinline__ void route_block(const Routing& a, int block,
                                            float* lds) {
  constexpr int NW = 4, TM = 16, RP = 16 * NT + 4;
  const int E = a.E, top = a.top, width = a.width, n_tok = a.n_tok;
  float* red = lds;
  float* logits = red + NW * TM * RP;
  float* choice = logits + TM * E;
  int* idx = (int*)(choice + NW * 2 * a.groups);
  float* wgt = (float*)(idx + TM * top);
  int* hist = (int*)(wgt + TM * top);
  int* base = hist + E;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & 63;
  const int n = lane & 15, g = lane >> 4;
  const int t0 = block * TM;
  const int left = n_tok - t0 < TM ? n_tok - t0 : TM;
  const bf16_t* hp =
      (const bf16_t*)a.h + (size_t)(t0 + (n < left ? n : left - 1)) * width;
  for (int e = tid; e < E; e += 256) hist[e] = 0;
  for (int e0 = 0; e0 < E; e0 += 16 * NT) {
    const bf16_t* wp[NT];
#pragma unroll
    for (int b = 0; b < NT; ++b) {
      const int e = e0 + b * 16 + n;
      wp[b] = (const bf16_t*)a.w + (size_t)(e < E ? e : E - 1) * width;
    }
    f32x4 acc[NT];
#pragma unroll
    for (int b = 0; b < NT; ++b) acc[b] = f32x4{0.f, 0.f, 0.f, 0.f};
    // CH pieces of 64 of the depth are in flight; past its end tokens
    // count as zero
    constexpr int CH = NT == 1 ? 4 : 2;
    for (int k0 = wave * 64; k0 < width; k0 += CH * NW * 64) {
      u32x4 hf[CH][2], wf[CH][2][NT];
#pragma unroll
      for (int c = 0; c < CH; ++c)
#pragma unroll
        for (int s = 0; s < 2; ++s) {
          const int k = k0 + c * NW * 64 + s * 32 + g * 8;
          const int kk = k < width ? k : 0;
          hf[c][s] = *reinterpret_cast<const u32x4*>(hp + kk);
#pragma unroll
          for (int b = 0; b < NT; ++b)
            wf[c][s][b] = *reinterpret_cast<const u32x4*>(wp[b] + kk);
        }
#pragma unroll
      for (int c = 0; c < CH; ++c)
#pragma unroll
        for (int s = 0; s < 2; ++s) {
          if (k0 + c * NW * 64 + s * 32 + g * 8 >= width)
            hf[c][s] = u32x4{0, 0, 0, 0};
#pragma unroll
          for (int b = 0; b < NT; ++b)
            acc[b] = mfma(wf[c][s][b], hf[c][s], acc[b]);
        }
    }
    // a lane holds experts 4g..4g+3 of token n
#pragma unroll
    for (int b = 0; b < NT; ++b)
      *reinterpret_cast<f32x4*>(
          &red[(wave * TM + n) * RP + b * 16 + g * 4]) = acc[b];
    __syncthreads();
    for (int i = tid; i < TM * 16 * NT; i += 256) {
      const int t = i / (16 * NT), e = i % (16 * NT);
      float x = 0.f;
#pragma unroll
      for (int v = 0; v < NW; ++v) x += red[(v * TM + t) * RP + e];
      if (e0 + e < E) logits[t * E + e0 + e] = x;
    }
    __syncthreads();
  }
  auto lanes = [&](auto size) {
    constexpr int L = decltype(size)::value;
    for (int i = tid / L; i < TM; i += 256 / L)
      if (i < left)
        choose_experts_lane<L>(
            tid % L < E ? logits[i * E + tid % L] : 0.f, E, top, a.groups,
            a.keep, a.scale, idx + i * top, wgt + i * top);
  };
  if (E <= 16) {
    lanes(std::integral_constant<int, 16>());
  } else if (E <= 32) {
    lanes(std::integral_constant<int, 32>());
  } else if (E <= 64) {
    lanes(std::integral_constant<int, 64>());
  } else {
    float* best = choice + wave * 2 * a.groups;
    for (int i = wave; i < left; i += NW) {
      choose_experts(logits + i * E, best, (int*)(best + a.groups), E, top,
                     a.groups, a.keep, a.scale, idx + i * top, wgt + i * top);
      __builtin_amdgcn_wave_barrier();
    }
  }
  __syncthreads();
  const int n_pairs = left * top;
  for (int i = tid; i < n_pairs; i += 256) {
    a.index[(size_t)t0 * top + i] = idx[i];
    a.weight[(size_t)t0 * top + i] = wgt[i];
  }
  if (!a.counts) return;
  // places in the experts' lists: one reservation an expert
  int* rank = (int*)red;
  for (int i = tid; i < n_pairs; i += 256)
    rank[i] = atomicAdd(&hist[idx[i]], 1);
  __syncthreads();
  for (int e = tid; e < E; e += 256)
    if (hist[e]) base[e] = atomicAdd(&a.counts[e], hist[e]);
  __syncthreads();
  for (int i = tid; i < n_pairs; i += 256)
    a.pairs[(size_t)idx[i] * n_tok + base[idx[i]] + rank[i]] = t0 * top + i;
}

// sizes that route_block takes
__host__ inline bool route_block_ok(const Routing& a, int dtype) {
  return dtype == 0 && a.width % 8 == 0 && a.E <= 256 && a.groups <= 64 &&
         a.top <= 32;
}
__host__ inline bool routing_ok(const Routing& a) {
  return a.width > 0 && a.E > 0 && a.E <= 1024 && a.groups > 0 &&
         a.E % a.groups == 0 && a.keep >= 1 && a.keep <= a.groups &&
         a.top >= 1 && a.top <= a.keep * (a.E / a.groups) &&
         (!a.counts || a.pairs) && (long long)a.n_tok * a.top < (1ll << 31);
}
