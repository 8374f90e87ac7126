// Matrix memory (see linear_scan.hip) of prompt portions on the matrix
// cores, 64 tokens at a time, bf16 storage.
//
// With F_t the sum of the chunk's log forget gates up to token t and m_in
// the running maximum before the chunk, m_t = max(F_t + m_in, b_t), b_t
// being the maximum of i_s + F_t - F_s over the chunk's s <= t.  Then
//   o_t   = q_t^T S_in exp(F_t + m_in - m_t)
//           + sum over s <= t of (q_t . k_s) exp(F_t - F_s + i_s - m_t) v_s,
//   S_out = exp(F + m_in - m) S_in
//           + sum over s of exp(F - F_s + i_s - m) k_s v_s^T  (F, m: the
//           last token's),
// and the normaliser is the same with v = 1: no exponent is above zero, and
// nothing is divided by a decay.
//
// q, k and v are bf16 as projected.  What is float, the weights of s and the
// state, enters a product as the sum of two bf16 numbers (relative error
// 2^-17); sums, the state and everything about the gates are float.
// Exponents are of two: F, c and b below carry log2(e).
#include "memory.h"
#include "mfma.h"

#define CHUNK 64

// Per token and head F, c = i - F and b, as gates [3][H][n_tok]; also
// copies normaliser and maximum out of the state to ``carry``
// [entries][H][extra_row(D)] (several workgroups read them later, and one
// replaces them).  A workgroup: a chunk and 16 heads, a wave each.
__global__ __launch_bounds__(1024) void memory_chunk_gates_kernel(
    float* __restrict__ gates, float* __restrict__ carry,
    const float* __restrict__ extra, const bf16_t* __restrict__ proj, int ld,
    int i_off, const float* __restrict__ bias, const int* __restrict__ e_start,
    const int* __restrict__ e_len, const int* __restrict__ e_pos,
    const int* __restrict__ e_row, int n_tok, int H, int D, float cap) {
  __shared__ float z[CHUNK][33];
  const int e = blockIdx.y, t0 = blockIdx.x * CHUNK, h0 = blockIdx.z * 16;
  const int len = e_len[e];
  if (t0 >= len) return;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & (WAVE - 1);
  const int heads = H - h0 < 16 ? H - h0 : 16;
  const size_t first = (size_t)e_start[e];
  if (t0 == 0) {
    const int row = extra_row(D);
    const bool resume = e_pos[e] > 0;
    const float* src = extra + ((size_t)e_row[e] * H + h0) * row;
    float* dst = carry + ((size_t)e * H + h0) * row;
    for (int i = tid; i < heads * row; i += 1024)
      dst[i] = resume ? src[i] : 0.f;
  }
  for (int i = tid; i < CHUNK * 32; i += 1024) {
    const int t = t0 + i / 32, c = i % 32, h = c % 16;
    if (h < heads)
      z[i / 32][c] =
          to_f(proj[(first + (t < len ? t : len - 1)) * ld + i_off +
                    c / 16 * H + h0 + h]);
  }
  __syncthreads();
  const int h = wave;
  if (h < heads) {
    float li, lf;
    memory_gates(z[lane][h] + bias[h0 + h], z[lane][16 + h] + bias[H + h0 + h],
                 cap, li, lf);
    float F = lf, b = li;
#pragma unroll
    for (int o = 1; o < WAVE; o <<= 1) {
      const float f1 = __shfl_up(F, o, WAVE), b1 = __shfl_up(b, o, WAVE);
      if (lane >= o) {
        b = fmaxf(b1 + F, b);
        F += f1;
      }
    }
    if (t0 + lane < len) {
      float* to = gates + (size_t)(h0 + h) * n_tok + first + t0 + lane;
      const size_t plane = (size_t)H * n_tok;
      to[0] = F * LOG2E;
      to[plane] = (li - F) * LOG2E;
      to[2 * plane] = b * LOG2E;
    }
  }
}

// two floats as sums of bf16 numbers, hi + lo
__device__ __forceinline__ void split2(float a, float b, unsigned& hi,
                                       unsigned& lo) {
  hi = to_bf16x2(a, b);
  lo = to_bf16x2(a - __uint_as_float(hi << 16),
                 b - __uint_as_float(hi & 0xffff0000u));
}

// One workgroup: VB value columns of one head of one entry, chunk after
// chunk.  Wave w has the chunk's queries 16 w .. 16 w + 15 and a quarter of
// the state's key channels, which it carries as floats; for the queries of
// all waves the state goes through LDS.  The next chunk is in flight
// meanwhile.
//   o [n_tok][H V]; state [slots][H][V][D]
template <int DQ, int VB>
__global__ __launch_bounds__(256, DQ <= 128 ? 2 : 1)
void memory_chunk_kernel(
    float* __restrict__ o, float* __restrict__ state,
    float* __restrict__ extra, const bf16_t* __restrict__ proj, int ld,
    int k_off, int v_off, const float* __restrict__ gates,
    const float* __restrict__ carry, const int* __restrict__ e_start,
    const int* __restrict__ e_len, const int* __restrict__ e_pos,
    const int* __restrict__ e_row, int n_tok, int H, int D, int V,
    float q_scale) {
  constexpr int KD = DQ / 32, VT = VB / 16, DT = DQ < 64 ? 1 : DQ / 64;
  constexpr int KP = DQ + 8, VP = VB + 8;       // LDS pitches
  constexpr int KL = DQ / 32, VL = VB / 32;     // pieces of a tile a thread
  __shared__ unsigned short lk[CHUNK * KP];
  __shared__ unsigned short lv[CHUNK * VP];
  // [2][VB + 1][KP]: the columns of S and n, high and low parts
  extern __shared__ __attribute__((aligned(16))) unsigned short ls[];
  __shared__ __attribute__((aligned(16))) float lc[CHUNK], lw[CHUNK];
  constexpr int LO = (VB + 1) * KP;
  const int e = blockIdx.y;
  const int head = blockIdx.x % H, c0 = blockIdx.x / H * VB;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & (WAVE - 1);
  const int n = lane & 15, g = lane >> 4;
  const int len = e_len[e];
  const size_t first = (size_t)e_start[e];
  const bool resume = e_pos[e] > 0;
  const bf16_t* rows = proj + first * ld;
  const float* gate = gates + (size_t)head * n_tok + first;
  const size_t plane = (size_t)H * n_tok;
  const int d0 = wave * DT * 16;      // the wave's key channels
  const bool holds = DQ >= 64 || d0 < DQ;  // 32 channels are two waves'
  float* sp = state + ((size_t)e_row[e] * H + head) * V * D;
  const float* cr = carry + ((size_t)e * H + head) * extra_row(D);

  // the state: S[dt][v] holds key channels d0 + 16 dt + 4 g .. + 3 of
  // column 16 v + n, N[dt] the normaliser's
  f32x4 S[DT][VT], N[DT];
#pragma unroll
  for (int a = 0; a < DT; ++a) {
    const int d = d0 + a * 16 + g * 4;
    const bool real = holds && d < D;
    N[a] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (real) {
      const float4 x = *reinterpret_cast<const float4*>(cr + d);
      N[a] = f32x4{x.x, x.y, x.z, x.w};
    }
#pragma unroll
    for (int v = 0; v < VT; ++v) {
      const int col = c0 + v * 16 + n;
      S[a][v] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (resume && real && col < V) {
        const float4 x =
            *reinterpret_cast<const float4*>(sp + (size_t)col * D + d);
        S[a][v] = f32x4{x.x, x.y, x.z, x.w};
      }
    }
  }
  float m = cr[extra_row(D) - 4] * LOG2E;

  auto share = [&]() {  // the state for all waves' queries
    if (!holds) return;
#pragma unroll
    for (int a = 0; a < DT; ++a) {
      const int d = d0 + a * 16 + g * 4;
#pragma unroll
      for (int v = 0; v < VT; ++v) {
        uint2 hi, lo;
        split2(S[a][v][0], S[a][v][1], hi.x, lo.x);
        split2(S[a][v][2], S[a][v][3], hi.y, lo.y);
        unsigned short* to = ls + (v * 16 + n) * KP + d;
        *reinterpret_cast<uint2*>(to) = hi;
        *reinterpret_cast<uint2*>(to + LO) = lo;
      }
      if (n == 0) {
        uint2 hi, lo;
        split2(N[a][0], N[a][1], hi.x, lo.x);
        split2(N[a][2], N[a][3], hi.y, lo.y);
        *reinterpret_cast<uint2*>(ls + VB * KP + d) = hi;
        *reinterpret_cast<uint2*>(ls + LO + VB * KP + d) = lo;
      }
    }
  };
  share();

  // Columns past D meet zeros of the query, those past V are dropped: what
  // stands for them is finite, and of the size of the others.
  u32x4 pk[KL], pv[VL], qn[KD];
  float gf, gc, gb;  // of token ``lane`` of the chunk
  auto fetch = [&](int t0) {
    const int end = len - 1 - t0;  // the entry's last token
    const bf16_t* at = rows + (size_t)t0 * ld;
#pragma unroll
    for (int i = 0; i < KL; ++i) {
      const int p = tid + i * 256, t = p / (DQ / 8), d = p % (DQ / 8) * 8;
      pk[i] = *reinterpret_cast<const u32x4*>(
          at + (unsigned)((t < end ? t : end) * ld + k_off + head * D +
                          (d < D ? d : 0)));
    }
#pragma unroll
    for (int i = 0; i < VL; ++i) {
      const int p = tid + i * 256, t = p / (VB / 8), d = p % (VB / 8) * 8;
      pv[i] = *reinterpret_cast<const u32x4*>(
          at + (unsigned)((t < end ? t : end) * ld + v_off + head * V + c0 +
                          (c0 + d < V ? d : 0)));
    }
    const int tq = wave * 16 + n;
#pragma unroll
    for (int k = 0; k < KD; ++k) {
      const int d = k * 32 + g * 8;
      qn[k] = *reinterpret_cast<const u32x4*>(
          at + (unsigned)((tq < end ? tq : end) * ld + head * D +
                          (d < D ? d : 0)));
    }
    const float* x = gate + t0 + (lane < end ? lane : end);
    gf = x[0];
    gc = x[plane];
    gb = x[2 * plane];
  };
  fetch(0);

  for (int t0 = 0; t0 < len; t0 += CHUNK) {
#pragma unroll
    for (int i = 0; i < KL; ++i) {
      const int p = tid + i * 256;
      *reinterpret_cast<u32x4*>(
          &lk[p / (DQ / 8) * KP + p % (DQ / 8) * 8]) = pk[i];
    }
#pragma unroll
    for (int i = 0; i < VL; ++i) {
      const int p = tid + i * 256;
      *reinterpret_cast<u32x4*>(
          &lv[p / (VB / 8) * VP + p % (VB / 8) * 8]) = pv[i];
    }
    u32x4 qf[KD];
#pragma unroll
    for (int k = 0; k < KD; ++k)
      qf[k] = k * 32 + g * 8 < D ? qn[k] : u32x4{0, 0, 0, 0};
    // past the entry's end nothing is forgotten and nothing comes in
    if (t0 + lane >= len) gc = -INFINITY;
    const float mt = fmaxf(gf + m, gb);
    const float f_end = __shfl(gf, 63, WAVE), m_end = __shfl(mt, 63, WAVE);
    const float decay = __builtin_amdgcn_exp2f(f_end + m - m_end);
    if (wave == 0) {
      lc[lane] = gc;
      lw[lane] = __builtin_amdgcn_exp2f(f_end + gc - m_end);
    }
    // of this lane's query
    const float f_q = __shfl(gf, wave * 16 + n, WAVE);
    const float m_q = __shfl(mt, wave * 16 + n, WAVE);
    const float from = __builtin_amdgcn_exp2f(f_q + m - m_q);
    const float least = __builtin_amdgcn_exp2f(-m_q);
    m = m_end;
    __syncthreads();
    if (t0 + CHUNK < len) fetch(t0 + CHUNK);

    // scores with the chunk's keys, weighted (all of them: the wave of the
    // last queries needs them all, and the others wait for it)
    f32x4 s[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) s[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < KD; ++k)
#pragma unroll
      for (int t = 0; t < 4; ++t)
        s[t] = mfma(*reinterpret_cast<const u32x4*>(
                        &lk[(t * 16 + n) * KP + k * 32 + g * 8]),
                    qf[k], s[t]);
    u32x4 hi[2], lo[2];
    float den = 0.f;
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      const float4 c = *reinterpret_cast<const float4*>(&lc[t * 16 + g * 4]);
      const float cs[4] = {c.x, c.y, c.z, c.w};
      const int age = (wave - t) * 16 + n - g * 4;  // of key (t, 0)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float w = s[t][i] * __builtin_amdgcn_exp2f(f_q - m_q + cs[i]);
        s[t][i] = age >= i ? w : 0.f;
        den += s[t][i];
      }
      unsigned h0, h1, l0, l1;
      split2(s[t][0], s[t][1], h0, l0);
      split2(s[t][2], s[t][3], h1, l1);
      hi[t / 2][t % 2 * 2] = h0;
      hi[t / 2][t % 2 * 2 + 1] = h1;
      lo[t / 2][t % 2 * 2] = l0;
      lo[t / 2][t % 2 * 2 + 1] = l1;
    }
    den += __shfl_xor(den, 16, WAVE);
    den += __shfl_xor(den, 32, WAVE);

    // what the state before the chunk gives
    f32x4 acc[VT], nq = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int v = 0; v < VT; ++v) acc[v] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < KD; ++k) {
      const unsigned short* r = ls + k * 32 + g * 8;
#pragma unroll
      for (int v = 0; v < VT; ++v) {
        const unsigned short* x = r + (v * 16 + n) * KP;
        acc[v] = mfma(*reinterpret_cast<const u32x4*>(x), qf[k], acc[v]);
        acc[v] = mfma(*reinterpret_cast<const u32x4*>(x + LO), qf[k], acc[v]);
      }
      const unsigned short* x = r + VB * KP;  // the same for every row
      nq = mfma(*reinterpret_cast<const u32x4*>(x), qf[k], nq);
      nq = mfma(*reinterpret_cast<const u32x4*>(x + LO), qf[k], nq);
    }
#pragma unroll
    for (int v = 0; v < VT; ++v) acc[v] *= from;
#pragma unroll
    for (int a = 0; a < DT; ++a) {
      N[a] *= decay;
#pragma unroll
      for (int v = 0; v < VT; ++v) S[a][v] *= decay;
    }

    // the chunk's values into the outputs and the state
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int r = p * 32 + g * 4;  // keys r .. + 3 and r + 16 .. + 3
      u32x4 vf[VT];
#pragma unroll
      for (int v = 0; v < VT; ++v)
        vf[v] = load_columns(
            &lv[(r + (n >> 2)) * VP + v * 16 + (n & 3) * 4], 16 * VP);
#pragma unroll
      for (int v = 0; v < VT; ++v) {
        acc[v] = mfma(vf[v], hi[p], acc[v]);
        acc[v] = mfma(vf[v], lo[p], acc[v]);
      }
      if (holds) {
        const float4 wa = *reinterpret_cast<const float4*>(&lw[r]);
        const float4 wb = *reinterpret_cast<const float4*>(&lw[r + 16]);
        const float ws[8] = {wa.x, wa.y, wa.z, wa.w, wb.x, wb.y, wb.z, wb.w};
        const u32x4 one = {0x3f803f80u, 0x3f803f80u, 0x3f803f80u,
                           0x3f803f80u};
#pragma unroll
        for (int a = 0; a < DT; ++a) {
          const u32x4 kf = load_columns(
              &lk[(r + (n >> 2)) * KP + d0 + a * 16 + (n & 3) * 4], 16 * KP);
          u32x4 kh, kl;
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            unsigned h, l;
            split2(__uint_as_float(kf[i] << 16) * ws[2 * i],
                   __uint_as_float(kf[i] & 0xffff0000u) * ws[2 * i + 1], h,
                   l);
            kh[i] = h;
            kl[i] = l;
          }
#pragma unroll
          for (int v = 0; v < VT; ++v) {
            S[a][v] = mfma(kh, vf[v], S[a][v]);
            S[a][v] = mfma(kl, vf[v], S[a][v]);
          }
          N[a] = mfma(kh, one, N[a]);
          N[a] = mfma(kl, one, N[a]);
        }
      }
    }

    const int t = t0 + wave * 16 + n;
    if (t < len) {
      den = fabsf((den + nq[0] * from) * q_scale);
      const float f = q_scale / (fmaxf(den, least) + MEMORY_EPS);
      float* dst = o + ((first + t) * H + head) * V + c0;
#pragma unroll
      for (int v = 0; v < VT; ++v) {
        const int d = v * 16 + g * 4;
        if (c0 + d < V)  // V is a multiple of 8
          *reinterpret_cast<float4*>(dst + d) =
              make_float4(acc[v][0] * f, acc[v][1] * f, acc[v][2] * f,
                          acc[v][3] * f);
      }
    }
    __syncthreads();
    if (t0 + CHUNK < len) share();
  }

  if (!holds) return;
  float* ex = extra + ((size_t)e_row[e] * H + head) * extra_row(D);
#pragma unroll
  for (int a = 0; a < DT; ++a) {
    const int d = d0 + a * 16 + g * 4;
    if (d >= D) continue;
#pragma unroll
    for (int v = 0; v < VT; ++v) {
      const int col = c0 + v * 16 + n;
      if (col < V)
        *reinterpret_cast<float4*>(sp + (size_t)col * D + d) = make_float4(
            S[a][v][0], S[a][v][1], S[a][v][2], S[a][v][3]);
    }
    if (c0 == 0 && n == 0)
      *reinterpret_cast<float4*>(ex + d) =
          make_float4(N[a][0], N[a][1], N[a][2], N[a][3]);
  }
  if (c0 == 0 && tid == 0) ex[extra_row(D) - 4] = m / LOG2E;
}

extern "C" {

int hy_memory_chunk(void* o, void* gates, void* carry, void* state,
                    void* extra, const void* proj, int ld, int k_off,
                    int v_off, int i_off, const void* bias,
                    const void* e_start, const void* e_len, const void* e_pos,
                    const void* e_row, int n_entries, int max_len, int n_tok,
                    int H, int D, int V, float q_scale, float cap,
                    void* stream) {
  if (H <= 0 || D <= 0 || V <= 0 || D % 8 || V % 8 || D > 256 || ld % 8 ||
      k_off % 8 || v_off % 8 || n_entries > 65535 || !(cap > 0.f))
    return -2;
  if (n_entries <= 0 || n_tok <= 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  hipLaunchKernelGGL(
      memory_chunk_gates_kernel,
      dim3((max_len + CHUNK - 1) / CHUNK, n_entries, (H + 15) / 16),
      dim3(1024), 0, s, (float*)gates, (float*)carry, (const float*)extra,
      (const bf16_t*)proj, ld, i_off, (const float*)bias,
      (const int*)e_start, (const int*)e_len, (const int*)e_pos,
      (const int*)e_row, n_tok, H, D, cap);
  HY_CHECK();
#define GO(DQ, VB)                                                           \
  do {                                                                       \
    constexpr int lds = 2 * (VB + 1) * (DQ + 8) * 2;                         \
    static const hipError_t ready = hipFuncSetAttribute(                     \
        reinterpret_cast<const void*>(memory_chunk_kernel<DQ, VB>),          \
        hipFuncAttributeMaxDynamicSharedMemorySize, lds);                    \
    if (ready != hipSuccess) return -3;                                      \
    hipLaunchKernelGGL((memory_chunk_kernel<DQ, VB>),                        \
                       dim3(H * ((V + VB - 1) / VB), n_entries), dim3(256),  \
                       lds, s, (float*)o, (float*)state, (float*)extra,      \
                       (const bf16_t*)proj, ld, k_off, v_off,                \
                       (const float*)gates, (const float*)carry,             \
                       (const int*)e_start, (const int*)e_len,               \
                       (const int*)e_pos, (const int*)e_row, n_tok, H, D, V, \
                       q_scale);                                             \
  } while (0)
#define PICK(DQ)                \
  do {                          \
    if (wide) GO(DQ, 64);       \
    else GO(DQ, 32);            \
  } while (0)
  // 64 columns a workgroup where that still fills the chip
  const bool wide = (long long)n_entries * H * ((V + 63) / 64) >= 256;
  if (D <= 32) PICK(32);
  else if (D <= 64) PICK(64);
  else if (D <= 128) PICK(128);
  else PICK(256);
#undef PICK
#undef GO
  HY_CHECK();
  return 0;
}

}  // extern "C"
