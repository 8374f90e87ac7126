// Matrix-core forms of windowed and chunked grouped-query attention (see
// window_attention.hip for the masks, the gate and the cache layout), bf16 storage, float softmax.
//
//  * window_flash_kernel   prompts: 128 rows a workgroup, a row being one
//    head of one query; all heads of a key/value head are rows side by
//    side, so that a staged tile serves as many of them as there are.
//  * window_decode_kernel  single tokens: all heads of a key/value head
//    against each cached row read once; window_merge_kernel joins the
//    parts where keys are split.
//
// Both compute S^T = K Q^T with 16x16x32 MFMAs: a lane holds, for ONE row
// n = lane % 16, the scores of keys 4g..4g+3 of each 16-key tile
// (g = lane / 16).
#include "paged_tiles.h"

// ---------------------------------------------------------------------------
// Prompt portions: 32 rows a wave, tiles of 64 keys through LDS, the next
// tile in registers.
//   item = (packed query, query position, queries, table row)
template <int DQ, int DV>
__global__ __launch_bounds__(256, DQ + DV <= 256 ? 2 : 1)
void window_flash_kernel(
    bf16_t* __restrict__ out, int ld_out, const bf16_t* __restrict__ proj,
    int ld, int g_off, const bf16_t* __restrict__ cache,
    const int* __restrict__ items, const int* __restrict__ bt, int max_blocks,
    int H, int G, int D, int V, Mask mask) {
  constexpr int KD = DQ / 32, VT = DV / 16;
  using St = Stage<1, DQ, DV>;
  __shared__ unsigned short lk[64 * St::KP];
  __shared__ unsigned short lv[64 * St::VP];
  const int kv = blockIdx.x % G, R = H / G;
  const int* it = items + blockIdx.x / G * 4;
  const int q_row = it[0], q_pos = it[1], n_rows = it[2] * R;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & 63;
  const int n = lane & 15, g = lane >> 4;
  const int last = q_pos + it[2] - 1;

  int qi[2], at[2], span[2];  // this lane's queries, heads, keys before
  u32x4 qf[2][KD];
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    int r = wave * 32 + a * 16 + n;
    r = r < n_rows ? r : n_rows - 1;
    qi[a] = r / R;
    at[a] = kv * R + r - qi[a] * R;
    span[a] = mask.span(q_pos + qi[a]);
    const bf16_t* q =
        proj + (size_t)(q_row + qi[a]) * ld + (size_t)at[a] * D;
#pragma unroll
    for (int k = 0; k < KD; ++k) {
      const int d = k * 32 + g * 8;
      qf[a][k] = d < D ? *reinterpret_cast<const u32x4*>(q + d)
                       : u32x4{0, 0, 0, 0};
    }
  }
  // positions of the wave's first and last query
  const int w_lo = q_pos + wave * 32 / R;
  const int w_hi = q_pos + (wave * 32 + 31) / R;
  // and the first keys they see
  const int w_lo_key = w_lo - mask.span(w_lo);
  const int w_hi_key = w_hi - mask.span(w_hi);
  const int lo = mask.first(q_pos) & ~(PAGE - 1);

  St st(cache, bt + (size_t)it[3] * max_blocks, G, kv, D, V, last);
  u32x4 pk[St::KL], pv[St::VL];
  int pg[4];
  f32x4 o[2][VT];
  float m[2], l[2];
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    m[a] = -1e30f;
    l[a] = 0.f;
#pragma unroll
    for (int v = 0; v < VT; ++v) o[a][v] = f32x4{0.f, 0.f, 0.f, 0.f};
  }

  st.fetch_pages(lo, pg);
  st.fetch(lo, pg, pk, pv);
  if (lo + 64 <= last) st.fetch_pages(lo + 64, pg);
  for (int j0 = lo; j0 <= last; j0 += 64) {
    St::store(lk, lv, pk, pv);
    __syncthreads();
    if (j0 + 64 <= last) {
      st.fetch(j0 + 64, pg, pk, pv);
      if (j0 + 128 <= last) st.fetch_pages(j0 + 128, pg);
    }
    // a tile none of the wave's queries sees is skipped
    if (j0 <= w_hi && j0 + 63 >= w_lo_key) {
      f32x4 s[2][4];
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        s[0][t] = s[1][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < KD; ++k) {
          const u32x4 kf = *reinterpret_cast<const u32x4*>(
              &lk[(t * 16 + n) * St::KP + k * 32 + g * 8]);
          s[0][t] = mfma(kf, qf[0][k], s[0][t]);
          s[1][t] = mfma(kf, qf[1][k], s[1][t]);
        }
      }
      const bool whole = j0 + 63 <= w_lo && j0 >= w_hi_key;
      u32x4 pf[2][2];
#pragma unroll
      for (int a = 0; a < 2; ++a) {
        if (!whole) {
          const int age = q_pos + qi[a] - j0 - g * 4;
#pragma unroll
          for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int i = 0; i < 4; ++i)
              s[a][t][i] =
                  (unsigned)(age - t * 16 - i) <= (unsigned)span[a]
                      ? s[a][t][i]
                      : -INFINITY;
        }
        float mx = m[a];
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
          for (int i = 0; i < 4; ++i) mx = fmaxf(mx, s[a][t][i]);
        mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
        mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
        const float keep = __builtin_amdgcn_exp2f(m[a] - mx);
        m[a] = mx;
        float sum = 0.f;
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const float p = __builtin_amdgcn_exp2f(s[a][t][i] - mx);
            s[a][t][i] = p;
            sum += p;
          }
        l[a] = l[a] * keep + sum;
#pragma unroll
        for (int v = 0; v < VT; ++v) o[a][v] *= keep;
#pragma unroll
        for (int p = 0; p < 2; ++p)
          pf[a][p] = u32x4{to_bf16x2(s[a][2 * p][0], s[a][2 * p][1]),
                           to_bf16x2(s[a][2 * p][2], s[a][2 * p][3]),
                           to_bf16x2(s[a][2 * p + 1][0], s[a][2 * p + 1][1]),
                           to_bf16x2(s[a][2 * p + 1][2], s[a][2 * p + 1][3])};
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
    float sum = l[a];
    sum += __shfl_xor(sum, 16, WAVE);
    sum += __shfl_xor(sum, 32, WAVE);
    if (wave * 32 + a * 16 + n >= n_rows) continue;
    const size_t tok = q_row + qi[a];
    float f = 1.f / sum;
    if (g_off >= 0)
      f = 1.f / (sum * (1.f + __expf(-to_f(proj[tok * ld + g_off + at[a]]))));
    bf16_t* dst = out + tok * ld_out + (size_t)at[a] * V;
#pragma unroll
    for (int v = 0; v < VT; ++v) {
      const int d = v * 16 + g * 4;
      if (d < V)
        *reinterpret_cast<uint2*>(dst + d) =
            make_uint2(to_bf16x2(o[a][v][0] * f, o[a][v][1] * f),
                       to_bf16x2(o[a][v][2] * f, o[a][v][3] * f));
    }
  }
}

// ---------------------------------------------------------------------------
// Single tokens.  One workgroup: one query, up to 16 heads of one
// key/value head, one part of its window.  Each wave scores 16 of a
// tile's 64 keys, the weights go through LDS, and each wave accumulates a
// quarter of the value columns.
//   acc [N][H][parts][V], ml [N][H][parts] (maximum, sum); one part: the
//   output itself
template <int DQ, int DV>
__global__ __launch_bounds__(256, 2)
void window_decode_kernel(
    bf16_t* __restrict__ out, int ld_out, float* __restrict__ ws_acc,
    float* __restrict__ ws_ml, const bf16_t* __restrict__ proj, int ld,
    int g_off, const bf16_t* __restrict__ cache,
    const int* __restrict__ pos_, const int* __restrict__ row_,
    const int* __restrict__ bt, int max_blocks, int H, int G, int D, int V,
    Mask mask, int parts) {
  constexpr int KD = DQ / 32, NV = DV / 64, PP = 64 + 8;
  using St = Stage<1, DQ, DV>;
  __shared__ unsigned short lk[64 * St::KP];
  __shared__ unsigned short lv[64 * St::VP];
  __shared__ unsigned short lp[16 * PP];
  __shared__ float lmax[16][4], lsum[16][4];
  const int q = blockIdx.x, part = blockIdx.z;
  const int R = H / G, ht = (R + 15) / 16;
  const int kv = blockIdx.y / ht, h0 = blockIdx.y % ht * 16;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & 63;
  const int n = lane & 15, g = lane >> 4;
  const int pos = pos_[q];
  const int h = kv * R + h0 + n;  // this lane's head
  const bool real = h0 + n < R;

  const int span = mask.span(pos);
  const int lo = mask.first(pos) & ~(PAGE - 1);
  const int tiles = (pos - lo) / 64 + 1;
  const int per = (tiles + parts - 1) / parts;
  const int t_lo = part * per;
  const int t_hi = t_lo + per < tiles ? t_lo + per : tiles;

  St st(cache, bt + (size_t)row_[q] * max_blocks, G, kv, D, V, pos);
  u32x4 pk[St::KL], pv[St::VL];
  int pg[4];
  if (t_lo < t_hi) {
    st.fetch_pages(lo + t_lo * 64, pg);
    st.fetch(lo + t_lo * 64, pg, pk, pv);
    if (t_lo + 1 < t_hi) st.fetch_pages(lo + t_lo * 64 + 64, pg);
  }
  u32x4 qf[KD];
#pragma unroll
  for (int k = 0; k < KD; ++k) {
    const int d = k * 32 + g * 8;
    qf[k] = u32x4{0, 0, 0, 0};
    if (d < D && real)
      qf[k] = *reinterpret_cast<const u32x4*>(proj + (size_t)q * ld +
                                              (size_t)h * D + d);
  }
  // what the sum is multiplied with to gate
  float z = 1.f;
  if (real && g_off >= 0)
    z += __expf(-to_f(proj[(size_t)q * ld + g_off + h]));

  f32x4 o[NV];
  float m = -1e30f, l = 0.f;
#pragma unroll
  for (int v = 0; v < NV; ++v) o[v] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int t = t_lo; t < t_hi; ++t) {
    St::store(lk, lv, pk, pv);
    __syncthreads();
    if (t + 1 < t_hi) {
      st.fetch(lo + t * 64 + 64, pg, pk, pv);
      if (t + 2 < t_hi) st.fetch_pages(lo + t * 64 + 128, pg);
    }
    const int j = lo + t * 64 + wave * 16 + g * 4;
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < KD; ++k)
      s = mfma(*reinterpret_cast<const u32x4*>(
                   &lk[(wave * 16 + n) * St::KP + k * 32 + g * 8]),
               qf[k], s);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      s[i] = (unsigned)(pos - j - i) <= (unsigned)span ? s[i] : -INFINITY;
    float mx = fmaxf(fmaxf(s[0], s[1]), fmaxf(s[2], s[3]));
    mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
    mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
    if (g == 0) lmax[n][wave] = mx;
    __syncthreads();
    mx = m;
#pragma unroll
    for (int i = 0; i < 4; ++i) mx = fmaxf(mx, lmax[n][i]);
    const float keep = __builtin_amdgcn_exp2f(m - mx);
    m = mx;
    l *= keep;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      s[i] = __builtin_amdgcn_exp2f(s[i] - m);
      l += s[i];
    }
    *reinterpret_cast<uint2*>(&lp[n * PP + wave * 16 + g * 4]) =
        make_uint2(to_bf16x2(s[0], s[1]), to_bf16x2(s[2], s[3]));
    __syncthreads();
#pragma unroll
    for (int v = 0; v < NV; ++v) o[v] *= keep;
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const u32x4 pf = *reinterpret_cast<const u32x4*>(
          &lp[n * PP + ks * 32 + g * 8]);
#pragma unroll
      for (int v = 0; v < NV; ++v)
        o[v] = mfma(load_columns(&lv[(ks * 32 + g * 8 + (n >> 2)) * St::VP +
                                     (wave * NV + v) * 16 + (n & 3) * 4],
                                 4 * St::VP),
                    pf, o[v]);
    }
    __syncthreads();
  }
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  if (g == 0) lsum[n][wave] = l;
  __syncthreads();
  if (!real) return;
  l = lsum[n][0] + lsum[n][1] + lsum[n][2] + lsum[n][3];
  if (parts == 1) {
    const float f = 1.f / (l * z);
    bf16_t* dst = out + (size_t)q * ld_out + (size_t)h * V;
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int d = (wave * NV + v) * 16 + g * 4;
      if (d < V)
        *reinterpret_cast<uint2*>(dst + d) =
            make_uint2(to_bf16x2(o[v][0] * f, o[v][1] * f),
                       to_bf16x2(o[v][2] * f, o[v][3] * f));
    }
    return;
  }
  const size_t at = ((size_t)q * H + h) * parts + part;
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int d = (wave * NV + v) * 16 + g * 4;
    if (d < V)
      *reinterpret_cast<float4*>(ws_acc + at * V + d) =
          make_float4(o[v][0], o[v][1], o[v][2], o[v][3]);
  }
  if (wave == 0 && g == 0) {
    ws_ml[at * 2] = m;
    ws_ml[at * 2 + 1] = l;
  }
}

// Join the parts and gate.  One wave a head; lane p first holds part p's
// weight.  A part without keys has sum 0 and the lowest maximum.
#define PARTS_MAX 64
__global__ __launch_bounds__(256) void window_merge_kernel(
    bf16_t* __restrict__ out, int ld_out, const float* __restrict__ ws_acc,
    const float* __restrict__ ws_ml, const bf16_t* __restrict__ proj, int ld,
    int g_off, int H, int V, int parts) {
  const int q = blockIdx.x, h = blockIdx.y * 4 + threadIdx.x / WAVE;
  if (h >= H) return;
  const int lane = threadIdx.x & 63;
  const size_t at = ((size_t)q * H + h) * parts;
  const int c = lane * 4;  // V <= 256 columns
  const float z = g_off < 0 ? 0.f : to_f(proj[(size_t)q * ld + g_off + h]);
  float m = -1e30f, w = 0.f;
  if (lane < parts) {
    const float2 ml =
        *reinterpret_cast<const float2*>(ws_ml + (at + lane) * 2);
    m = ml.x;
    w = ml.y;
  }
  float mx = m;
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, WAVE));
  const float f = __builtin_amdgcn_exp2f(m - mx);
  const float gate = g_off < 0 ? 1.f : 1.f + __expf(-z);
  w = f / (wave_sum(w * f) * gate);

  float o[4] = {0.f, 0.f, 0.f, 0.f};
  const float* src = ws_acc + at * V + (c < V ? c : 0);
#pragma unroll 8
  for (int i = 0; i < parts; ++i) {
    const float wi = __shfl(w, i, WAVE);
    float x[4];
    load4(src + (size_t)i * V, x);
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] += x[j] * wi;
  }
  if (c < V) store4(out + (size_t)q * ld_out + (size_t)h * V + c, o);
}

static bool window_ok(int ld, int ld_out, int H, int G, int D, int V,
                      int window) {
  return G > 0 && H > 0 && H % G == 0 && D > 0 && V > 0 && D % 8 == 0 &&
         V % 8 == 0 && D <= 256 && V <= 256 && ld % 8 == 0 &&
         ld_out % 8 == 0 && window >= 1;
}

// GO(DQ, DV) for the smallest tile that holds D and V
#define WINDOW_SIZES(D, V)                               \
  do {                                                   \
    if (D <= 32) { constexpr int Q = 32; WINDOW_V(V); }  \
    else if (D <= 64) { constexpr int Q = 64; WINDOW_V(V); } \
    else if (D <= 96) { constexpr int Q = 96; WINDOW_V(V); } \
    else if (D <= 128) { constexpr int Q = 128; WINDOW_V(V); } \
    else { constexpr int Q = 256; WINDOW_V(V); }         \
  } while (0)
#define WINDOW_V(V)                                      \
  do {                                                   \
    if (V <= 64) GO(Q, 64);                              \
    else if (V <= 128) GO(Q, 128);                       \
    else GO(Q, 256);                                     \
  } while (0)

extern "C" {

int hy_window_flash(void* out, int ld_out, const void* proj, int ld,
                    int g_off, const void* cache, const void* items,
                    int n_items, const void* bt, int max_blocks, int H, int G,
                    int D, int V, int window, int chunk, void* stream) {
  if (!window_ok(ld, ld_out, H, G, D, V, window) || H / G > 128) return -2;
  if (n_items <= 0) return 0;
  const Mask mask{window, chunk != 0};
#define GO(DQ, DV)                                                           \
  hipLaunchKernelGGL((window_flash_kernel<DQ, DV>),                          \
                     dim3((unsigned)n_items * G), dim3(256), 0,              \
                     (hipStream_t)stream, (bf16_t*)out, ld_out,              \
                     (const bf16_t*)proj, ld, g_off, (const bf16_t*)cache,   \
                     (const int*)items, (const int*)bt, max_blocks, H, G, D, \
                     V, mask)
  WINDOW_SIZES(D, V);
#undef GO
  HY_CHECK();
  return 0;
}

int hy_window_decode(void* out, int ld_out, void* acc, void* ml,
                     const void* proj, int ld, int g_off, const void* cache,
                     const void* pos, const void* row, const void* bt,
                     int max_blocks, int H, int G, int D, int V, int window,
                     int chunk, int n_rows, int parts, void* stream) {
  if (!window_ok(ld, ld_out, H, G, D, V, window) || parts < 1 ||
      parts > PARTS_MAX || (parts > 1 && (!acc || !ml)))
    return -2;
  if (n_rows <= 0) return 0;
  const int tiles = (H / G + 15) / 16;
  if (G * tiles > 65535) return -2;
  const Mask mask{window, chunk != 0};
#define GO(DQ, DV)                                                           \
  hipLaunchKernelGGL((window_decode_kernel<DQ, DV>),                         \
                     dim3(n_rows, G * tiles, parts), dim3(256), 0,           \
                     (hipStream_t)stream, (bf16_t*)out, ld_out, (float*)acc, \
                     (float*)ml, (const bf16_t*)proj, ld, g_off,             \
                     (const bf16_t*)cache, (const int*)pos, (const int*)row, \
                     (const int*)bt, max_blocks, H, G, D, V, mask, parts)
  WINDOW_SIZES(D, V);
#undef GO
  HY_CHECK();
  if (parts == 1) return 0;
  hipLaunchKernelGGL(window_merge_kernel, dim3(n_rows, (H + 3) / 4),
                     dim3(256), 0, (hipStream_t)stream, (bf16_t*)out, ld_out,
                     (const float*)acc, (const float*)ml,
                     (const bf16_t*)proj, ld, g_off, H, V, parts);
  HY_CHECK();
  return 0;
}

}  // extern "C"
