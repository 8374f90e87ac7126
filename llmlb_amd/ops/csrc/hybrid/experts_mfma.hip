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

// 64 lanes copy 16 bytes each from their own addresses to 1 KB of LDS from
// byte ``to`` on.  The copy counts as a load of the wave; nothing but
// wait_barrier waits for it.
__device__ __forceinline__ void copy_to_lds(const bf16_t* src, unsigned to) {
  asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off"
               ::"s"(__builtin_amdgcn_readfirstlane(to)), "v"(src)
               : "memory");
}
__device__ __forceinline__ unsigned lds_byte(const unsigned short* p) {
  return (unsigned)(uintptr_t)(
      (const __attribute__((address_space(3))) unsigned short*)p);
}
// All but the newest N copies and loads of the wave are done, and its LDS
// reads; then the workgroup's barrier.
template <int N>
__device__ __forceinline__ void wait_barrier() {
  asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)\n\ts_barrier" ::"n"(N)
               : "memory");
}

// LDS rows are P pieces of 16 bytes; piece c of row r lies at
// c ^ swizzle(r), so that lanes reading one piece of the rows of an
// operand meet different banks.
template <int P>
__device__ __forceinline__ int swizzle_in(int r) {
  return P == 8 ? r & 7 : (r >> 1) & 3;
}
template <int P>
__device__ __forceinline__ int swizzle_w(int r) {
  return P == 8 ? (r & 3) | ((r >> 1) & 4) : ((r >> 1) & 1) | ((r >> 2) & 2);
}

// Workgroup: BM pairs x BN outputs, WM x WN waves; BK of the depth a step.
// LDS holds ST steps, the copies of a step start ST - 1 steps ahead.
// Within 32 outputs of a wave, row g * 8 + t * 4 + i of the matrix is row
// 4 g + i of MFMA tile t: a lane then holds 8 consecutive outputs of each
// of its pairs.
template <int BM, int BN, int WM, int WN, int BK, int ST>
__global__ __launch_bounds__(WM * WN * 64, WM * WN == 4 ? 2 : 1)
void expert_tile_kernel(
    bf16_t* __restrict__ out, const bf16_t* __restrict__ in,
    const bf16_t* __restrict__ w, const int* __restrict__ counts,
    const int* __restrict__ pairs, int E, int N, int K, int div, int act,
    int n_tok, int n_blocks) {
  constexpr int NW = WM * WN, TM = BM / WM / 16, TN = BN / WN / 64;
  constexpr int P = BK / 8, RC = 64 / P;  // pieces of a row, rows of a copy
  constexpr int CA = BM / RC / NW, CB = BN / RC / NW;  // copies a wave
  constexpr int C = CA + CB, SIZE = (BM + BN) * BK;
  __shared__ __align__(1024) unsigned short lds[ST * SIZE];
  __shared__ ExpertTiles<BM> tiles;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int n = lane & 15, g = lane >> 4;
  if (wave == 0) tiles.count(counts, E);
  __syncthreads();
  // neighbouring tiles on one XCD, which gets every eighth workgroup
  const int whole = tiles.whole[E - 1] * n_blocks;
  const int rest = tiles.rest[E - 1] * n_blocks;
  const int per = (whole + 7) / 8, rest_per = (rest + 7) / 8;
  const int xcd = blockIdx.x & 7, local = blockIdx.x >> 3;
  const bool is_rest = local >= per;
  const int id = is_rest ? xcd * rest_per + local - per : xcd * per + local;
  if (is_rest ? local - per >= rest_per || id >= rest : id >= whole) return;
  const ExpertTile t = tiles.get(counts, E, id / n_blocks, is_rest);
  const int n0 = id % n_blocks * BN;
  const int* list = pairs + (size_t)t.expert * n_tok + t.first;
  const bf16_t* we = w + (size_t)t.expert * N * K;

  const bf16_t *ap[CA], *bp[CB];
  int ac[CA], bc[CB];  // the lane's column within a row
#pragma unroll
  for (int i = 0; i < CA; ++i) {
    const int r = (wave * CA + i) * RC + lane / P;
    ac[i] = ((lane % P) ^ swizzle_in<P>(r)) * 8;
    ap[i] = in + (size_t)(list[r < t.n ? r : t.n - 1] / div) * K + ac[i];
  }
#pragma unroll
  for (int i = 0; i < CB; ++i) {
    const int r = (wave * CB + i) * RC + lane / P;
    bc[i] = ((lane % P) ^ swizzle_w<P>(r)) * 8;
    bp[i] = we + (size_t)(n0 + r < N ? n0 + r : N - 1) * K + bc[i];
  }
  const unsigned base = lds_byte(lds);
  const bf16_t* zero = reinterpret_cast<const bf16_t*>(zero_piece);
  // past the depth zeros are copied: every step has as many copies
  auto fetch = [&](int k0, int place) {
    const unsigned to = base + place * SIZE * 2;
#pragma unroll
    for (int i = 0; i < CA; ++i)
      copy_to_lds(k0 + ac[i] < K ? ap[i] + k0 : zero,
                  to + (wave * CA + i) * 1024);
#pragma unroll
    for (int i = 0; i < CB; ++i)
      copy_to_lds(k0 + bc[i] < K ? bp[i] + k0 : zero,
                  to + BM * BK * 2 + (wave * CB + i) * 1024);
  };
  const int wm = wave / WN * (BM / WM), wn = wave % WN * (BN / WN);
  f32x4 acc[TM][TN][4];
#pragma unroll
  for (int a = 0; a < TM; ++a)
#pragma unroll
    for (int b = 0; b < TN; ++b)
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[a][b][i] = f32x4{0.f, 0.f, 0.f, 0.f};

  // the lane's numbers of a place, before the row tile and MFMA step
  const int ra = wm + n, rb = wn + (n >> 2) * 8 + (n & 3);
#pragma unroll
  for (int s = 0; s < ST - 1; ++s) fetch(s * BK, s);
  // One barrier a step: past it, every wave has read the place of the step
  // before, which the newest copies take.
  int place = 0, free = ST - 1;
  for (int k0 = 0; k0 < K; k0 += BK) {
    wait_barrier<(ST - 2) * C>();
    fetch(k0 + (ST - 1) * BK, free);
    __builtin_amdgcn_sched_barrier(0);
    const unsigned short* st = lds + place * SIZE;
    free = place;
    place = place + 1 == ST ? 0 : place + 1;
    if (wm >= t.n || n0 + wn >= N) continue;  // nothing for this wave
#pragma unroll
    for (int s = 0; s < BK / 32; ++s) {
      const unsigned short* pa =
          st + ra * BK + ((s * 4 + g) ^ swizzle_in<P>(ra)) * 8;
      const unsigned short* pb =
          st + BM * BK + rb * BK + ((s * 4 + g) ^ swizzle_w<P>(rb)) * 8;
      // the pieces of rows 4 further lie elsewhere where P is 8
      const unsigned short* pb4 =
          st + BM * BK + (rb + 4) * BK +
          ((s * 4 + g) ^ swizzle_w<P>(rb + 4)) * 8;
      u32x4 af[TM], bf[TN][4];
#pragma unroll
      for (int a = 0; a < TM; ++a)
        af[a] = *reinterpret_cast<const u32x4*>(pa + a * 16 * BK);
#pragma unroll
      for (int b = 0; b < TN; ++b)
#pragma unroll
        for (int i = 0; i < 4; ++i)
          bf[b][i] = *reinterpret_cast<const u32x4*>(
              (i & 1 ? pb4 : pb) + (b * 64 + (i >> 1) * 32) * BK);
#pragma unroll
      for (int a = 0; a < TM; ++a)
#pragma unroll
        for (int b = 0; b < TN; ++b)
#pragma unroll
          for (int i = 0; i < 4; ++i)
            acc[a][b][i] = mfma(bf[b][i], af[a], acc[a][b][i]);
    }
  }
  // no copy is under way when the workgroup's LDS is given back
  wait_barrier<0>();
#pragma unroll
  for (int a = 0; a < TM; ++a) {
    const int r = wm + a * 16 + n;
    if (r >= t.n) continue;
    bf16_t* dst = out + (size_t)list[r] * N;
#pragma unroll
    for (int b = 0; b < TN; ++b) {
      const int c = n0 + wn + b * 64 + g * 8;
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
        if (c + i * 32 < N)
          __builtin_nontemporal_store(
              u32x4{x[4 * i], x[4 * i + 1], x[4 * i + 2], x[4 * i + 3]},
              reinterpret_cast<u32x4*>(dst + c + i * 32));
    }
  }
}

// Few pairs: workgroup (expert, 16 NT outputs), the depth split over its
// four waves.
#define FEW_PAIRS 2048  // most that fit a workgroup's list
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
  // CH pieces of 64 of the depth are in flight; past its end inputs count
  // as zero
  constexpr int CH = 2;
  for (int k0 = wave * 64; k0 < K; k0 += CH * 256) {
    u32x4 wf[CH][2][NT], xf[CH][2][MT];
#pragma unroll
    for (int c = 0; c < CH; ++c)
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        const int k = k0 + c * 256 + s * 32 + g * 8;
        const int kk = k < K ? k : 0;
#pragma unroll
        for (int b = 0; b < NT; ++b)
          wf[c][s][b] = *reinterpret_cast<const u32x4*>(wp[b] + kk);
#pragma unroll
        for (int a = 0; a < MT; ++a)
          xf[c][s][a] = *reinterpret_cast<const u32x4*>(ip[a] + kk);
      }
#pragma unroll
    for (int c = 0; c < CH; ++c)
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        const bool inside = k0 + c * 256 + s * 32 + g * 8 < K;
#pragma unroll
        for (int a = 0; a < MT; ++a) {
          if (!inside) xf[c][s][a] = u32x4{0, 0, 0, 0};
#pragma unroll
          for (int b = 0; b < NT; ++b)
            acc[a][b] = mfma(wf[c][s][b], xf[c][s][a], acc[a][b]);
        }
      }
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

// tile: 0 128 x 128, 1 256 x 256, 2 128 x 256 (pairs x outputs)
int hy_expert_tiles(void* out, const void* in, const void* w,
                    const void* counts, const void* pairs, int E, int N,
                    int K, int div, int act, int n_tok, int n_pairs,
                    int tile, void* stream) {
  if (E <= 0 || E > EXPERTS_MAX || N <= 0 || K <= 0 || N % 8 || K % 8 ||
      div <= 0)
    return -2;
  if (n_tok <= 0 || n_pairs <= 0) return 0;
#define GO(BM, BN, WM, WN, BK, ST)                                                 \
  do {                                                                       \
    const long long nb = (N + BN - 1) / BN;                                  \
    const long long groups = (n_pairs / BM * nb + 7) / 8 +                   \
                             ((E < n_pairs ? E : n_pairs) * nb + 7) / 8;     \
    if (groups >= (1ll << 27)) return -2;                                    \
    hipLaunchKernelGGL((expert_tile_kernel<BM, BN, WM, WN, BK, ST>),                 \
                       dim3((unsigned)groups * 8),                           \
                       dim3(WM * WN * 64), 0, (hipStream_t)stream,           \
                       (bf16_t*)out, (const bf16_t*)in, (const bf16_t*)w,    \
                       (const int*)counts, (const int*)pairs, E, N, K, div,  \
                       act, n_tok, (int)nb);                                 \
  } while (0)
  switch (tile) {
    case 0: GO(128, 128, 2, 2, 64, 2); break;
    case 1: GO(256, 256, 4, 4, 64, 2); break;
    case 2: GO(128, 256, 2, 4, 32, 3); break;
    default: return -2;
  }
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
