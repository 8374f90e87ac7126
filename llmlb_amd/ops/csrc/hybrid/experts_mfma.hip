// Matrix-core products of tokens with their experts' matrices, bf16: for
// every (token, choice) pair p = token * top + choice
//   out[p] = act(w[expert] in[p / div]),  act(z) = max(z, 0)^2 or none.
//
//  * expert_tile_kernel  prompts: tiles of an expert's list (experts.h)
//    against tiles of its matrix, both copied to LDS directly
//  * expert_few_kernel   few pairs: a workgroup finds its expert's pairs
//    among all choices and streams some rows of its matrix once
//
// Both compute (w in^T) tiles: a lane holds outputs 4g..4g+3 (g = lane/16)
// of pair n = lane % 16.
#include "experts.h"
#include "mfma.h"

__device__ __align__(16) unsigned zero_piece[4];

// 64 lanes copy 16 bytes each from their own addresses to 1 KB of LDS
__device__ __forceinline__ void copy_to_lds(const bf16_t* src,
                                            unsigned short* dst) {
  __builtin_amdgcn_global_load_lds(
      (const __attribute__((address_space(1))) void*)src,
      (__attribute__((address_space(3))) void*)dst, 16, 0, 0);
}

// LDS rows are 64 numbers in 8 pieces of 16 bytes; piece c of row r lies
// at c ^ swizzle(r), so that lanes reading one piece of the rows of an
// operand meet different banks.
__device__ __forceinline__ int swizzle_in(int r) { return r & 7; }
__device__ __forceinline__ int swizzle_w(int r) {
  return (r & 3) | ((r >> 2) & 4);
}

// Workgroup: BM pairs x BN outputs, WM x WN waves.  Within 64 outputs of
// a wave, row g * 16 + t * 4 + i of the matrix is row 4 g + i of MFMA tile
// t: a lane then holds 16 consecutive outputs of each of its pairs.
template <int BM, int BN, int WM, int WN>
__global__ __launch_bounds__(WM * WN * 64) void expert_tile_kernel(
    bf16_t* __restrict__ out, const bf16_t* __restrict__ in,
    const bf16_t* __restrict__ w, const int* __restrict__ counts,
    const int* __restrict__ pairs, int E, int N, int K, int div, int act,
    int n_tok, int n_blocks, int m_blocks) {
  constexpr int NW = WM * WN, TM = BM / WM / 16, TN = BN / WN / 64;
  constexpr int CA = BM / 8 / NW, CB = BN / 8 / NW;  // copies a wave
  // two places for a step's tiles; variables of their own, so that reading
  // one is not taken to depend on copies to the other
  __shared__ unsigned short la0[BM * 64], la1[BM * 64];
  __shared__ unsigned short lb0[BN * 64], lb1[BN * 64];
  // neighbouring tiles on one XCD, which gets every eighth workgroup
  const int total = n_blocks * m_blocks, per = (total + 7) / 8;
  const int id = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
  if (id >= total) return;
  ExpertTile t;
  if (!find_tile<BM>(counts, E, id / n_blocks, t)) return;
  const int n0 = id % n_blocks * BN;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & 63;
  const int n = lane & 15, g = lane >> 4;
  const int* list = pairs + (size_t)t.expert * n_tok + t.first;
  const bf16_t* we = w + (size_t)t.expert * N * K;
  const bf16_t* zero = reinterpret_cast<const bf16_t*>(zero_piece);

  const bf16_t *ap[CA], *bp[CB];
  int ac[CA], bc[CB];  // the lane's column within a row
#pragma unroll
  for (int i = 0; i < CA; ++i) {
    const int r = (wave * CA + i) * 8 + (lane >> 3);
    ac[i] = ((lane & 7) ^ swizzle_in(r)) * 8;
    ap[i] = in + (size_t)(list[r < t.n ? r : t.n - 1] / div) * K + ac[i];
  }
#pragma unroll
  for (int i = 0; i < CB; ++i) {
    const int r = (wave * CB + i) * 8 + (lane >> 3);
    bc[i] = ((lane & 7) ^ swizzle_w(r)) * 8;
    bp[i] = we + (size_t)(n0 + r < N ? n0 + r : N - 1) * K + bc[i];
  }
  auto fetch = [&](int k0, unsigned short* la, unsigned short* lb) {
#pragma unroll
    for (int i = 0; i < CA; ++i)
      copy_to_lds(k0 + ac[i] < K ? ap[i] + k0 : zero,
                  &la[(wave * CA + i) * 512]);
#pragma unroll
    for (int i = 0; i < CB; ++i)
      copy_to_lds(k0 + bc[i] < K ? bp[i] + k0 : zero,
                  &lb[(wave * CB + i) * 512]);
  };
  const int wm = wave / WN * (BM / WM), wn = wave % WN * (BN / WN);
  f32x4 acc[TM][TN][4];
#pragma unroll
  for (int a = 0; a < TM; ++a)
#pragma unroll
    for (int b = 0; b < TN; ++b)
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[a][b][i] = f32x4{0.f, 0.f, 0.f, 0.f};

  // One barrier a step: past it, every wave has read the tile before this
  // one, whose place the next copy takes.
  auto step = [&](int k0, const unsigned short* la, const unsigned short* lb,
                  unsigned short* next_a, unsigned short* next_b) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (k0 + 64 < K) fetch(k0 + 64, next_a, next_b);
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      u32x4 af[TM], bf[TN][4];
#pragma unroll
      for (int a = 0; a < TM; ++a) {
        const int r = wm + a * 16 + n;
        af[a] = *reinterpret_cast<const u32x4*>(
            &la[r * 64 + ((s * 4 + g) ^ swizzle_in(r)) * 8]);
      }
#pragma unroll
      for (int b = 0; b < TN; ++b)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int r = wn + b * 64 + (n >> 2) * 16 + i * 4 + (n & 3);
          bf[b][i] = *reinterpret_cast<const u32x4*>(
              &lb[r * 64 + ((s * 4 + g) ^ swizzle_w(r)) * 8]);
        }
#pragma unroll
      for (int a = 0; a < TM; ++a)
#pragma unroll
        for (int b = 0; b < TN; ++b)
#pragma unroll
          for (int i = 0; i < 4; ++i)
            acc[a][b][i] = mfma(bf[b][i], af[a], acc[a][b][i]);
    }
  };
  fetch(0, la0, lb0);
  for (int k0 = 0; k0 < K; k0 += 128) {
    step(k0, la0, lb0, la1, lb1);
    if (k0 + 64 < K) step(k0 + 64, la1, lb1, la0, lb0);
  }
#pragma unroll
  for (int a = 0; a < TM; ++a) {
    const int r = wm + a * 16 + n;
    if (r >= t.n) continue;
    bf16_t* dst = out + (size_t)list[r] * N;
#pragma unroll
    for (int b = 0; b < TN; ++b) {
      const int c = n0 + wn + b * 64 + g * 16;
      unsigned x[8];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        f32x4 v = acc[a][b][i];
        if (act) {
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            v[j] = fmaxf(v[j], 0.f);
            v[j] *= v[j];
          }
        }
        x[2 * i] = to_bf16x2(v[0], v[1]);
        x[2 * i + 1] = to_bf16x2(v[2], v[3]);
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
        if (c + i * 8 < N)
          *reinterpret_cast<u32x4*>(dst + c + i * 8) = u32x4{
              x[4 * i], x[4 * i + 1], x[4 * i + 2], x[4 * i + 3]};
    }
  }
}

// Few pairs: workgroup (expert, 16 NT outputs), the depth split over its
// four waves.
#define FEW_PAIRS 2048
template <int MT, int NT>
__device__ __forceinline__ void expert_few_rows(
    bf16_t* __restrict__ out, const bf16_t* __restrict__ in,
    const bf16_t* (&wp)[NT], const unsigned short* list, int first, int count,
    float* red, int n0, int N, int K, int div, int act) {
  constexpr int RP = 16 * NT + 4;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & 63;
  const int n = lane & 15, g = lane >> 4;
  const bf16_t* ip[MT];
#pragma unroll
  for (int a = 0; a < MT; ++a) {
    const int r = first + a * 16 + n;
    ip[a] = in + (size_t)(list[r < count ? r : count - 1] / div) * K;
  }
  f32x4 acc[MT][NT];
#pragma unroll
  for (int a = 0; a < MT; ++a)
#pragma unroll
    for (int b = 0; b < NT; ++b) acc[a][b] = f32x4{0.f, 0.f, 0.f, 0.f};
  // 64 numbers of the depth at a time; past its end inputs count as zero
#pragma unroll 2
  for (int k0 = wave * 64; k0 < K; k0 += 256) {
    u32x4 wf[2][NT], xf[2][MT];
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const int k = k0 + s * 32 + g * 8;
      const bool inside = k < K;
      const int kk = inside ? k : 0;
#pragma unroll
      for (int b = 0; b < NT; ++b)
        wf[s][b] = *reinterpret_cast<const u32x4*>(wp[b] + kk);
#pragma unroll
      for (int a = 0; a < MT; ++a) {
        xf[s][a] = *reinterpret_cast<const u32x4*>(ip[a] + kk);
        if (!inside) xf[s][a] = u32x4{0, 0, 0, 0};
      }
    }
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int a = 0; a < MT; ++a)
#pragma unroll
        for (int b = 0; b < NT; ++b)
          acc[a][b] = mfma(wf[s][b], xf[s][a], acc[a][b]);
  }
#pragma unroll
  for (int a = 0; a < MT; ++a)
#pragma unroll
    for (int b = 0; b < NT; ++b)
      *reinterpret_cast<f32x4*>(
          &red[(wave * 16 * MT + a * 16 + n) * RP + b * 16 + g * 4]) =
          acc[a][b];
  __syncthreads();
  for (int i = tid; i < 16 * MT * 4 * NT; i += 256) {
    const int r = i / (4 * NT), c = i % (4 * NT) * 4;
    f32x4 x = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int v = 0; v < 4; ++v)
      x += *reinterpret_cast<const f32x4*>(
          &red[(v * 16 * MT + r) * RP + c]);
    if (act) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        x[j] = fmaxf(x[j], 0.f);
        x[j] *= x[j];
      }
    }
    if (first + r < count && n0 + c < N)
      *reinterpret_cast<uint2*>(out + (size_t)list[first + r] * N + n0 + c) =
          make_uint2(to_bf16x2(x[0], x[1]), to_bf16x2(x[2], x[3]));
  }
  __syncthreads();
}

template <int NT>
__global__ __launch_bounds__(256) void expert_few_kernel(
    bf16_t* __restrict__ out, const bf16_t* __restrict__ in,
    const bf16_t* __restrict__ w, const int* __restrict__ index, int N, int K,
    int div, int act, int n_pairs) {
  constexpr int MT = 4;
  __shared__ float red[4 * 16 * MT * (16 * NT + 4)];
  __shared__ unsigned short list[FEW_PAIRS];
  __shared__ int len;
  const int e = blockIdx.y, n0 = blockIdx.x * 16 * NT;
  const int tid = threadIdx.x;
  if (tid == 0) len = 0;
  __syncthreads();
  for (int p = tid; p < n_pairs; p += 256)
    if (index[p] == e) list[atomicAdd(&len, 1)] = (unsigned short)p;
  __syncthreads();
  const int count = len;
  if (count == 0) return;
  const bf16_t* wp[NT];
#pragma unroll
  for (int b = 0; b < NT; ++b) {
    const int r = n0 + b * 16 + (tid & 15);
    wp[b] = w + ((size_t)e * N + (r < N ? r : N - 1)) * K;
  }
#define ROWS(M)                                                             \
  expert_few_rows<M, NT>(out, in, wp, list, first, count, red, n0, N, K, div, \
                         act)
  for (int first = 0; first < count; first += 16 * MT) {
    const int left = count - first;
    if (left <= 16) ROWS(1);
    else if (left <= 32) ROWS(2);
    else ROWS(MT);
  }
#undef ROWS
}

extern "C" {

int hy_expert_tiles(void* out, const void* in, const void* w,
                    const void* counts, const void* pairs, int E, int N,
                    int K, int div, int act, int n_tok, int n_pairs,
                    void* stream) {
  if (E <= 0 || N <= 0 || K <= 0 || N % 8 || K % 8 || div <= 0) return -2;
  if (n_tok <= 0 || n_pairs <= 0) return 0;
#define GO(BM, BN, WM, WN)                                                   \
  do {                                                                       \
    const int m = n_pairs / BM + (E < n_pairs ? E : n_pairs);                \
    const int nb = (N + BN - 1) / BN;                                        \
    if ((long long)m * nb >= (1ll << 30)) return -2;                         \
    hipLaunchKernelGGL((expert_tile_kernel<BM, BN, WM, WN>),                 \
                       dim3((unsigned)(m * nb + 7) / 8 * 8),                 \
                       dim3(WM * WN * 64), 0, (hipStream_t)stream,           \
                       (bf16_t*)out, (const bf16_t*)in, (const bf16_t*)w,    \
                       (const int*)counts, (const int*)pairs, E, N, K, div,  \
                       act, n_tok, nb, m);                                   \
  } while (0)
  GO(128, 128, 2, 2);
#undef GO
  HY_CHECK();
  return 0;
}

int hy_expert_few(void* out, const void* in, const void* w, const void* index,
                  int E, int N, int K, int div, int act, int n_pairs,
                  void* stream) {
  if (E <= 0 || N <= 0 || K <= 0 || N % 8 || K % 8 || div <= 0 ||
      E > 65535 || n_pairs > FEW_PAIRS)
    return -2;
  if (n_pairs <= 0) return 0;
  hipLaunchKernelGGL((expert_few_kernel<2>), dim3((N + 31) / 32, E),
                     dim3(256), 0, (hipStream_t)stream, (bf16_t*)out,
                     (const bf16_t*)in, (const bf16_t*)w, (const int*)index,
                     N, K, div, act, n_pairs);
  HY_CHECK();
  return 0;
}

}  // extern "C"
