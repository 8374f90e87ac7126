// Matrix-core forms of differential attention (see pair_attention.hip for
// the cache layout), bf16 storage, float softmax.
//
//  * pair_flash_kernel   prompts: 64 queries of one head a workgroup.
//  * pair_decode_kernel  single tokens: all heads of a key/value head
//    against each cached row read once; pair_merge_kernel joins the parts.
//
// Both compute S^T = K Q^T with 16x16x32 MFMAs: a lane holds, for ONE query
// (or head) n = lane % 16, the scores of keys 4g..4g+3 of each 16-key tile
// (g = lane / 16).  In the prompt kernel the probabilities are then already
// laid out as the B operand of O^T = V^T P^T; V^T comes out of LDS through
// transposing reads.  Both maps share one staged V tile.
//
// Scores capped to |s| <= cap need no running maximum as long as
// exp(cap) times any sum of values stays in float's range: weights are then
// exp(s) itself (FIXED), for caps up to FIXED_CAP.
#include "paged_tiles.h"

#define FIXED_CAP 60.f

struct Capping {
  float to_z;      // score -> 2 log2(e) / cap * score (FIXED or capped)
  float cap_log2;  // cap log2(e), 0: no cap
};

// exp2 argument of a scaled score x (z = x * to_z already where capped)
__device__ __forceinline__ float cap_log2_of(float z, float cap_log2) {
  // cap tanh(s / cap) = cap - 2 cap / (1 + exp(2 s / cap))
  const float e = __builtin_amdgcn_exp2f(z);
  return cap_log2 - 2.f * cap_log2 * __builtin_amdgcn_rcpf(1.f + e);
}

// ---------------------------------------------------------------------------
// Prompt portions.  One workgroup: up to 64 queries of one head (16 a
// wave), tiles of 64 keys through LDS, the next tile in registers.
//   item = (packed query, query position, queries, table row)
template <int DQ, int DV, bool FIXED>
__global__ __launch_bounds__(256, DQ * 2 + DV <= 288 ? 2 : 1)
void pair_flash_kernel(
    bf16_t* __restrict__ out, int ld_out, const bf16_t* __restrict__ proj,
    int ld, int g_off, const bf16_t* __restrict__ cache,
    const int* __restrict__ items, const int* __restrict__ bt, int max_blocks,
    int H, int G, int D, int V, const float* __restrict__ q_scale,
    float to_z, float cap_log2, float lam, float gain, float eps) {
  constexpr int KD = DQ / 32, VT = DV / 16;
  using St = Stage<2, DQ, DV>;
  __shared__ unsigned short lk[64 * St::KP];
  __shared__ unsigned short lv[64 * St::VP];
  const int* it = items + (blockIdx.x / H) * 4;
  int h = blockIdx.x % H;
  if (H % 8 == 0)  // neighbouring heads on one XCD: its L2 serves them
    h = (h & 7) * (H / 8) + (h >> 3);
  const int q_row = it[0], q_pos = it[1], n_q = it[2];
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & 63;
  const int n = lane & 15, g = lane >> 4;
  const int last = q_pos + n_q - 1;

  const int mine = wave * 16 + n;  // this lane's query
  const int r = mine < n_q ? mine : n_q - 1;
  u32x4 qf[2][KD];
#pragma unroll
  for (int a = 0; a < 2; ++a)
#pragma unroll
    for (int k = 0; k < KD; ++k) {
      const int d = k * 32 + g * 8;
      qf[a][k] = u32x4{0, 0, 0, 0};
      if (d < D)
        qf[a][k] = *reinterpret_cast<const u32x4*>(
            proj + (size_t)(q_row + r) * ld + (size_t)(h * 2 + a) * D + d);
    }
  const float scale = q_scale[q_pos + r] * to_z;

  St st(cache, bt + (size_t)it[3] * max_blocks, G, h / (H / G), D, V, last);
  u32x4 pk[St::KL], pv[St::VL];
  int pg[4];
  f32x4 o[2][VT];
  float m[2], l[2];
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    m[a] = FIXED ? 0.f : -1e30f;
    l[a] = 0.f;
#pragma unroll
    for (int v = 0; v < VT; ++v) o[a][v] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const int w_lo = q_pos + wave * 16, w_hi = w_lo + 15;

  st.fetch_pages(0, pg);
  st.fetch(0, pg, pk, pv);
  if (64 <= last) st.fetch_pages(64, pg);
  for (int j0 = 0; j0 <= last; j0 += 64) {
    St::store(lk, lv, pk, pv);
    __syncthreads();
    if (j0 + 64 <= last) {
      st.fetch(j0 + 64, pg, pk, pv);
      if (j0 + 128 <= last) st.fetch_pages(j0 + 128, pg);
    }
    if (j0 <= w_hi) {  // a tile none of the wave's queries sees is skipped
      const bool whole = j0 + 63 <= w_lo;
      u32x4 pf[2][2];
#pragma unroll
      for (int a = 0; a < 2; ++a) {
        f32x4 s[4];
#pragma unroll
        for (int t = 0; t < 4; ++t) {
          s[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int k = 0; k < KD; ++k)
            s[t] = mfma(*reinterpret_cast<const u32x4*>(
                            &lk[(t * 16 + n) * St::KP + a * DQ + k * 32 +
                                g * 8]),
                        qf[a][k], s[t]);
        }
        float mx = m[a];
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            float x = s[t][i] * scale;
            if (FIXED || cap_log2 > 0.f) x = cap_log2_of(x, cap_log2);
            s[t][i] = x;
          }
        if (!whole) {
          const int age = q_pos + mine - j0 - g * 4;
#pragma unroll
          for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int i = 0; i < 4; ++i)
              s[t][i] = age - t * 16 - i >= 0 ? s[t][i] : -INFINITY;
        }
        if (!FIXED) {
#pragma unroll
          for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int i = 0; i < 4; ++i) mx = fmaxf(mx, s[t][i]);
          mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
          mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
          const float keep = __builtin_amdgcn_exp2f(m[a] - mx);
          m[a] = mx;
          l[a] *= keep;
#pragma unroll
          for (int v = 0; v < VT; ++v) o[a][v] *= keep;
        }
        float sum = 0.f;
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const float p =
                __builtin_amdgcn_exp2f(FIXED ? s[t][i] : s[t][i] - mx);
            s[t][i] = p;
            sum += p;
          }
        l[a] += sum;
#pragma unroll
        for (int p = 0; p < 2; ++p)
          pf[a][p] = u32x4{to_bf16x2(s[2 * p][0], s[2 * p][1]),
                           to_bf16x2(s[2 * p][2], s[2 * p][3]),
                           to_bf16x2(s[2 * p + 1][0], s[2 * p + 1][1]),
                           to_bf16x2(s[2 * p + 1][2], s[2 * p + 1][3])};
      }
#pragma unroll
      for (int v = 0; v < VT; ++v)
#pragma unroll
        for (int p = 0; p < 2; ++p) {
          const u32x4 vf = load_columns(
              &lv[(p * 32 + g * 4 + (n >> 2)) * St::VP + v * 16 +
                  (n & 3) * 4],
              16 * St::VP);
          o[0][v] = mfma(vf, pf[0][p], o[0][v]);
          o[1][v] = mfma(vf, pf[1][p], o[1][v]);
        }
    }
    __syncthreads();
  }
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    l[a] += __shfl_xor(l[a], 16, WAVE);
    l[a] += __shfl_xor(l[a], 32, WAVE);
  }
  const float i1 = 1.f / l[0], i2 = lam / l[1];
  float ssq = 0.f;
#pragma unroll
  for (int v = 0; v < VT; ++v) {
    o[0][v] = o[0][v] * i1 - o[1][v] * i2;
#pragma unroll
    for (int i = 0; i < 4; ++i) ssq += o[0][v][i] * o[0][v][i];
  }
  ssq += __shfl_xor(ssq, 16, WAVE);  // columns past V hold zeros
  ssq += __shfl_xor(ssq, 32, WAVE);
  const float rn = gain / sqrtf(ssq / V + eps);
  if (mine >= n_q) return;
  const bf16_t* gate =
      proj + (size_t)(q_row + mine) * ld + g_off + (size_t)h * V;
  bf16_t* dst = out + (size_t)(q_row + mine) * ld_out + (size_t)h * V;
#pragma unroll
  for (int v = 0; v < VT; ++v) {
    const int d = v * 16 + g * 4;
    if (d >= V) continue;
    float z[4], x[4];
    load4(gate + d, z);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      x[i] = o[0][v][i] * rn / (1.f + __expf(-z[i]));
    store4(dst + d, x);
  }
}

// ---------------------------------------------------------------------------
// Single tokens.  One workgroup: one query, up to 16 heads of one
// key/value head, one part of its keys.  Each wave scores 16 of a tile's
// 64 keys for both maps, the weights go through LDS, and each wave
// accumulates a quarter of the value columns.
//   acc [N][H][2][parts][V], ml the same with (maximum, sum)
template <int DQ, int DV, bool FIXED>
__global__ __launch_bounds__(256, 2)
void pair_decode_kernel(
    float* __restrict__ ws_acc, float* __restrict__ ws_ml,
    const bf16_t* __restrict__ proj, int ld, const bf16_t* __restrict__ cache,
    const int* __restrict__ pos_, const int* __restrict__ row_,
    const int* __restrict__ bt, int max_blocks, int H, int G, int D, int V,
    const float* __restrict__ q_scale, float to_z, float cap_log2,
    int parts) {
  constexpr int KD = DQ / 32, NV = DV / 64, PP = 64 + 8;
  using St = Stage<2, DQ, DV>;
  __shared__ unsigned short lk[64 * St::KP];
  __shared__ unsigned short lv[64 * St::VP];
  __shared__ unsigned short lp[2][16 * PP];
  __shared__ float lmax[2][16][4], lsum[2][16][4];
  const int q = blockIdx.x, part = blockIdx.z;
  const int R = H / G, ht = (R + 15) / 16;
  const int kv = blockIdx.y / ht, h0 = blockIdx.y % ht * 16;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & 63;
  const int n = lane & 15, g = lane >> 4;
  const int pos = pos_[q];
  const int h = kv * R + h0 + n;  // this lane's head
  const bool real = h0 + n < R;

  const int tiles = pos / 64 + 1;
  const int per = (tiles + parts - 1) / parts;
  const int t_lo = part * per;
  const int t_hi = t_lo + per < tiles ? t_lo + per : tiles;

  St st(cache, bt + (size_t)row_[q] * max_blocks, G, kv, D, V, pos);
  u32x4 pk[St::KL], pv[St::VL];
  int pg[4];
  if (t_lo < t_hi) {
    st.fetch_pages(t_lo * 64, pg);
    st.fetch(t_lo * 64, pg, pk, pv);
    if (t_lo + 1 < t_hi) st.fetch_pages(t_lo * 64 + 64, pg);
  }
  u32x4 qf[2][KD];
#pragma unroll
  for (int a = 0; a < 2; ++a)
#pragma unroll
    for (int k = 0; k < KD; ++k) {
      const int d = k * 32 + g * 8;
      qf[a][k] = u32x4{0, 0, 0, 0};
      if (d < D && real)
        qf[a][k] = *reinterpret_cast<const u32x4*>(
            proj + (size_t)q * ld + (size_t)(h * 2 + a) * D + d);
    }
  const float scale = q_scale[pos] * to_z;

  f32x4 o[2][NV];
  float m[2], l[2];
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    m[a] = FIXED ? 0.f : -1e30f;
    l[a] = 0.f;
#pragma unroll
    for (int v = 0; v < NV; ++v) o[a][v] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  for (int t = t_lo; t < t_hi; ++t) {
    St::store(lk, lv, pk, pv);
    __syncthreads();
    if (t + 1 < t_hi) {
      st.fetch(t * 64 + 64, pg, pk, pv);
      if (t + 2 < t_hi) st.fetch_pages(t * 64 + 128, pg);
    }
    const int j = t * 64 + wave * 16 + g * 4;
    f32x4 s[2];
#pragma unroll
    for (int a = 0; a < 2; ++a) {
      s[a] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KD; ++k)
        s[a] = mfma(*reinterpret_cast<const u32x4*>(
                        &lk[(wave * 16 + n) * St::KP + a * DQ + k * 32 +
                            g * 8]),
                    qf[a][k], s[a]);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        float x = s[a][i] * scale;
        if (FIXED || cap_log2 > 0.f) x = cap_log2_of(x, cap_log2);
        s[a][i] = j + i <= pos ? x : -INFINITY;
      }
    }
    float keep[2];
    if (!FIXED) {
#pragma unroll
      for (int a = 0; a < 2; ++a) {
        float mx = fmaxf(fmaxf(s[a][0], s[a][1]), fmaxf(s[a][2], s[a][3]));
        mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
        mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
        if (g == 0) lmax[a][n][wave] = mx;
      }
      __syncthreads();
#pragma unroll
      for (int a = 0; a < 2; ++a) {
        float x = m[a];
#pragma unroll
        for (int i = 0; i < 4; ++i) x = fmaxf(x, lmax[a][n][i]);
        keep[a] = __builtin_amdgcn_exp2f(m[a] - x);
        m[a] = x;
        l[a] *= keep[a];
      }
    }
#pragma unroll
    for (int a = 0; a < 2; ++a) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        s[a][i] =
            __builtin_amdgcn_exp2f(FIXED ? s[a][i] : s[a][i] - m[a]);
        l[a] += s[a][i];
      }
      *reinterpret_cast<uint2*>(&lp[a][n * PP + wave * 16 + g * 4]) =
          make_uint2(to_bf16x2(s[a][0], s[a][1]),
                     to_bf16x2(s[a][2], s[a][3]));
    }
    __syncthreads();
    if (!FIXED) {
#pragma unroll
      for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int v = 0; v < NV; ++v) o[a][v] *= keep[a];
    }
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      u32x4 pf[2];
#pragma unroll
      for (int a = 0; a < 2; ++a)
        pf[a] = *reinterpret_cast<const u32x4*>(
            &lp[a][n * PP + ks * 32 + g * 8]);
#pragma unroll
      for (int v = 0; v < NV; ++v) {
        const u32x4 vf = load_columns(
            &lv[(ks * 32 + g * 8 + (n >> 2)) * St::VP +
                (wave * NV + v) * 16 + (n & 3) * 4],
            4 * St::VP);
        o[0][v] = mfma(vf, pf[0], o[0][v]);
        o[1][v] = mfma(vf, pf[1], o[1][v]);
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    l[a] += __shfl_xor(l[a], 16, WAVE);
    l[a] += __shfl_xor(l[a], 32, WAVE);
    if (g == 0) lsum[a][n][wave] = l[a];
  }
  __syncthreads();
  if (!real) return;
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    const size_t at = (((size_t)q * H + h) * 2 + a) * parts + part;
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int d = (wave * NV + v) * 16 + g * 4;
      if (d < V)
        *reinterpret_cast<float4*>(ws_acc + at * V + d) =
            make_float4(o[a][v][0], o[a][v][1], o[a][v][2], o[a][v][3]);
    }
    if (wave == 0 && g == 0) {
      ws_ml[at * 2] = m[a];
      ws_ml[at * 2 + 1] = lsum[a][n][0] + lsum[a][n][1] + lsum[a][n][2] +
                          lsum[a][n][3];
    }
  }
}

// Join the parts of both maps, subtract, norm, gate.  One wave a head;
// lane a 32 + p first holds the weight of map a's part p.
#define PARTS_MAX 32
__global__ __launch_bounds__(256) void pair_merge_kernel(
    bf16_t* __restrict__ out, int ld_out, const float* __restrict__ ws_acc,
    const float* __restrict__ ws_ml, const bf16_t* __restrict__ proj, int ld,
    int g_off, int H, int V, int parts, float lam, float gain, float eps) {
  const int q = blockIdx.x, h = blockIdx.y * 4 + threadIdx.x / WAVE;
  if (h >= H) return;
  const int lane = threadIdx.x & 63;
  const size_t at = ((size_t)q * H + h) * 2 * parts;
  const int c = lane * 4;  // V <= 256 columns
  float z[4] = {0.f, 0.f, 0.f, 0.f};
  if (c < V) load4(proj + (size_t)q * ld + g_off + (size_t)h * V + c, z);
  float m = -1e30f, w = 0.f;
  const int a = lane >> 5, p = lane & 31;
  if (p < parts) {
    const float2 ml =
        *reinterpret_cast<const float2*>(ws_ml + (at + a * parts + p) * 2);
    m = ml.x;
    w = ml.y;
  }
  float mx = m;
#pragma unroll
  for (int o = 16; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, WAVE));
  const float f = __builtin_amdgcn_exp2f(m - mx);
  float sum = w * f;
#pragma unroll
  for (int o = 16; o > 0; o >>= 1) sum += __shfl_xor(sum, o, WAVE);
  w = f * (a == 0 ? 1.f : -lam) / sum;

  float o[4] = {0.f, 0.f, 0.f, 0.f};
  const float* src = ws_acc + at * V + (c < V ? c : 0);
#pragma unroll 8
  for (int i = 0; i < 2 * parts; ++i) {
    const float wi = __shfl(w, i < parts ? i : 32 + i - parts, WAVE);
    float x[4];
    load4(src + (size_t)i * V, x);
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] += x[j] * wi;
  }
  const float ssq =
      c < V ? o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3] : 0.f;
  const float rn = gain / sqrtf(wave_sum(ssq) / V + eps);
  if (c >= V) return;
#pragma unroll
  for (int j = 0; j < 4; ++j) o[j] *= rn / (1.f + __expf(-z[j]));
  store4(out + (size_t)q * ld_out + (size_t)h * V + c, o);
}

static bool pair_ok(int ld, int ld_out, int g_off, int H, int G, int D,
                    int V) {
  return G > 0 && H > 0 && H % G == 0 && D > 0 && V > 0 && D % 8 == 0 &&
         V % 8 == 0 && D <= 128 && V <= 256 && ld % 8 == 0 &&
         ld_out % 8 == 0 && g_off % 8 == 0;
}

// GO(DQ, DV, FIXED) for the smallest tile that holds D and V
#define PAIR_SIZES(D, V, fixed)                          \
  do {                                                   \
    if (fixed) { constexpr bool F = true; PAIR_D(D, V); } \
    else { constexpr bool F = false; PAIR_D(D, V); }     \
  } while (0)
#define PAIR_D(D, V)                                     \
  do {                                                   \
    if (D <= 32) { constexpr int Q = 32; PAIR_V(V); }    \
    else if (D <= 64) { constexpr int Q = 64; PAIR_V(V); } \
    else { constexpr int Q = 128; PAIR_V(V); }           \
  } while (0)
#define PAIR_V(V)                                        \
  do {                                                   \
    if (V <= 64) GO(Q, 64, F);                           \
    else if (V <= 128) GO(Q, 128, F);                    \
    else GO(Q, 256, F);                                  \
  } while (0)

extern "C" {

int hy_pair_flash(void* out, int ld_out, const void* proj, int ld, int g_off,
                  const void* cache, const void* items, int n_items,
                  const void* bt, int max_blocks, int H, int G, int D, int V,
                  const void* q_scale, float cap, float lam, float gain,
                  float eps, void* stream) {
  if (!pair_ok(ld, ld_out, g_off, H, G, D, V)) return -2;
  if (n_items <= 0) return 0;
  const float to_z = cap > 0.f ? 2.f * LOG2E / cap : LOG2E;
#define GO(DQ, DV, FIXED)                                                    \
  hipLaunchKernelGGL((pair_flash_kernel<DQ, DV, FIXED>),                     \
                     dim3((unsigned)n_items * H), dim3(256), 0,              \
                     (hipStream_t)stream, (bf16_t*)out, ld_out,              \
                     (const bf16_t*)proj, ld, g_off, (const bf16_t*)cache,   \
                     (const int*)items, (const int*)bt, max_blocks, H, G, D, \
                     V, (const float*)q_scale, to_z, cap * LOG2E, lam, gain, \
                     eps)
  PAIR_SIZES(D, V, cap > 0.f && cap <= FIXED_CAP);
#undef GO
  HY_CHECK();
  return 0;
}

int hy_pair_decode(void* out, int ld_out, void* acc, void* ml,
                   const void* proj, int ld, int g_off, const void* cache,
                   const void* pos, const void* row, const void* bt,
                   int max_blocks, int H, int G, int D, int V,
                   const void* q_scale, float cap, float lam, float gain,
                   float eps, int n_rows, int parts, void* stream) {
  if (!pair_ok(ld, ld_out, g_off, H, G, D, V) || parts < 1 ||
      parts > PARTS_MAX)
    return -2;
  if (n_rows <= 0) return 0;
  const float to_z = cap > 0.f ? 2.f * LOG2E / cap : LOG2E;
  const int tiles = (H / G + 15) / 16;
  if (G * tiles > 65535) return -2;
#define GO(DQ, DV, FIXED)                                                    \
  hipLaunchKernelGGL((pair_decode_kernel<DQ, DV, FIXED>),                    \
                     dim3(n_rows, G * tiles, parts), dim3(256), 0,           \
                     (hipStream_t)stream, (float*)acc, (float*)ml,           \
                     (const bf16_t*)proj, ld, (const bf16_t*)cache,          \
                     (const int*)pos, (const int*)row, (const int*)bt,       \
                     max_blocks, H, G, D, V, (const float*)q_scale, to_z,    \
                     cap * LOG2E, parts)
  PAIR_SIZES(D, V, cap > 0.f && cap <= FIXED_CAP);
#undef GO
  HY_CHECK();
  hipLaunchKernelGGL(pair_merge_kernel, dim3(n_rows, (H + 3) / 4), dim3(256),
                     0, (hipStream_t)stream, (bf16_t*)out, ld_out,
                     (const float*)acc, (const float*)ml,
                     (const bf16_t*)proj, ld, g_off, H, V, parts, lam, gain,
                     eps);
  HY_CHECK();
  return 0;
}

}  // extern "C"
