// Matrix-core forms of latent attention, bf16 storage, float softmax.
//
//  * latent_flash_kernel   prompts: keys and values expanded from the
//    latents (library products), flash attention over a causal window.
//  * latent_decode_kernel  single tokens: the absorbed form, all heads of
//    a query against each latent row read once.
//
// Both compute S^T = K Q^T with 16x16x32 MFMAs: a lane then holds, for
// ONE query (or head) n = lane % 16, the scores of keys 4g..4g+3 of each
// 16-key tile (g = lane / 16).  Row maxima and sums stay within a lane
// and its three partners, rescaling factors are one scalar a lane, and in
// the prompt kernel the probabilities are already laid out as the B
// operand of O^T = V^T P^T (keys 4g+i of two tiles make one operand).
#include "mfma.h"

// ---------------------------------------------------------------------------
// Copy the latents that a portion's queries can see out of the pages, 16
// rows a workgroup: c [rows][rank], kr [rows][R].  ``blocks`` holds
// (table row, first key position, valid keys) per 64 rows; rows past the
// valid ones are zeroed.
__global__ __launch_bounds__(256) void latent_gather_kernel(
    bf16_t* __restrict__ c, bf16_t* __restrict__ kr,
    const bf16_t* __restrict__ cache, const int* __restrict__ blocks,
    const int* __restrict__ bt, int max_blocks, int rank, int R) {
  const int* blk = blocks + blockIdx.x / 4 * 3;
  const int row = blk[0], first = blk[1], valid = blk[2];
  const int pieces = (rank + R) / 8;
  const int r0 = blockIdx.x % 4 * 16;
#pragma unroll 4
  for (int i = threadIdx.x; i < 16 * pieces; i += 256) {
    const int r = r0 + i / pieces, d = (i % pieces) * 8;
    uint4 v = make_uint4(0, 0, 0, 0);
    if (r < valid)
      v = *reinterpret_cast<const uint4*>(
          cache + page_slot(bt, max_blocks, row, first + r) * (rank + R) + d);
    const size_t to = (size_t)(blockIdx.x / 4) * 64 + r;
    bf16_t* dst = d < rank ? c + to * rank + d : kr + to * R + (d - rank);
    *reinterpret_cast<uint4*>(dst) = v;
  }
}

// ---------------------------------------------------------------------------
// Flash attention of prompt portions.  One workgroup: 128 queries of one
// head (32 a wave), key tiles of 64 through LDS, the next tile in
// registers meanwhile.
//   item = (packed query row, query position, queries, key row, key
//           position of that row); key rows of an item are consecutive
//   q   = proj + h * (D + R), kx [keys][H D], kr [keys][R],
//   vt [H V][key_ld]  (values transposed), out [tokens][H V]
//   sink (null: none): a number per head whose power joins the sum
//   g_off >= 0: out times the sigmoid of proj's columns from there on
template <int DQ, int DV>
__global__ __launch_bounds__(256, DQ * 2 + DV <= 512 ? 2 : 1)
void latent_flash_kernel(
    bf16_t* __restrict__ out, const bf16_t* __restrict__ proj, int ld,
    const bf16_t* __restrict__ kx, const bf16_t* __restrict__ kr,
    const bf16_t* __restrict__ vt, int key_ld, const int* __restrict__ items,
    int H, int D, int R, int V, int window, float scale_log2,
    const float* __restrict__ sink, int g_off) {
  constexpr int KD = DQ / 32, VT = DV / 16;
  constexpr int KP = DQ + 8, VP = 64 + 8;  // LDS pitches
  constexpr int KL = 64 * DQ / 8 / 256, VL = DV * 64 / 8 / 256;
  __shared__ unsigned short lk[64 * KP];
  __shared__ unsigned short lv[DV * VP];
  const int h = blockIdx.x % H;
  const int* it = items + (blockIdx.x / H) * 5;
  const int q_row = it[0], q_pos = it[1], n_q = it[2], k_row = it[3],
            k_pos = it[4];
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & 63;
  const int n = lane & 15, g = lane >> 4;
  const int DR = D + R;

  // this wave's queries: 2 tiles of 16
  u32x4 qf[2][KD];
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    int r = wave * 32 + a * 16 + n;
    r = r < n_q ? r : n_q - 1;
    const bf16_t* q = proj + (size_t)(q_row + r) * ld + (size_t)h * DR;
#pragma unroll
    for (int k = 0; k < KD; ++k) {
      const int d = k * 32 + g * 8;
      qf[a][k] = d < DR ? *reinterpret_cast<const u32x4*>(q + d)
                        : u32x4{0, 0, 0, 0};
    }
  }

  // keys seen by this workgroup, as places in the item's key rows
  const int seen_lo = q_pos - window + 1 - k_pos;
  const int lo = (seen_lo > 0 ? seen_lo : 0) & ~63;
  const int hi = q_pos + n_q - k_pos;  // one past the last

  // the thread's pieces of a tile: pointers that move from tile to tile.
  // Columns past D + R meet a zero of the query, rows past V are dropped.
  u32x4 pk[KL], pv[VL];
  const bf16_t* k_src[KL];
  int k_step[KL];
  unsigned v_off[VL];
#pragma unroll
  for (int i = 0; i < KL; ++i) {
    const int p = tid + i * 256;
    const int d = (p % (DQ / 8)) * 8;
    const size_t key = (size_t)k_row + lo + p / (DQ / 8);
    const bool rotated = d >= D && R > 0;
    k_src[i] = rotated ? kr + key * R + (d < DR ? d - D : 0)
                       : kx + key * H * D + (size_t)h * D + (d < D ? d : 0);
    k_step[i] = 64 * (rotated ? R : H * D);
  }
#pragma unroll
  for (int i = 0; i < VL; ++i) {
    const int p = tid + i * 256;
    v_off[i] = (unsigned)(p / 8 < V ? p / 8 : V - 1) * key_ld + (p % 8) * 8;
  }
  const bf16_t* v_src = vt + (size_t)h * V * key_ld + k_row + lo;
  auto fetch = [&]() {
#pragma unroll
    for (int i = 0; i < KL; ++i) {
      pk[i] = *reinterpret_cast<const u32x4*>(k_src[i]);
      k_src[i] += k_step[i];
    }
#pragma unroll
    for (int i = 0; i < VL; ++i)
      pv[i] = *reinterpret_cast<const u32x4*>(v_src + v_off[i]);
    v_src += 64;
  };

  f32x4 o[2][VT];
  float m[2], l[2];
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    m[a] = sink ? sink[h] * LOG2E : -1e30f;
    l[a] = sink && g == 0 ? 1.f : 0.f;
#pragma unroll
    for (int v = 0; v < VT; ++v) o[a][v] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const int w_lo = q_pos + wave * 32 - k_pos;  // this wave's queries, as
  const int w_hi = w_lo + 31;                  // places in the key rows

  fetch();
  for (int j0 = lo; j0 < hi; j0 += 64) {
#pragma unroll
    for (int i = 0; i < KL; ++i) {
      const int p = tid + i * 256;
      *reinterpret_cast<u32x4*>(
          &lk[(p / (DQ / 8)) * KP + (p % (DQ / 8)) * 8]) = pk[i];
    }
#pragma unroll
    for (int i = 0; i < VL; ++i) {
      const int p = tid + i * 256;
      *reinterpret_cast<u32x4*>(&lv[(p / 8) * VP + (p % 8) * 8]) = pv[i];
    }
    __syncthreads();
    if (j0 + 64 < hi) fetch();
    // a tile none of the wave's queries sees costs nothing
    if (j0 <= w_hi && j0 + 63 > w_lo - window) {
      f32x4 s[2][4];
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        s[0][t] = s[1][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < KD; ++k) {
          const u32x4 kf = *reinterpret_cast<const u32x4*>(
              &lk[(t * 16 + n) * KP + k * 32 + g * 8]);
          s[0][t] = mfma(kf, qf[0][k], s[0][t]);
          s[1][t] = mfma(kf, qf[1][k], s[1][t]);
        }
      }
      const bool whole = j0 + 63 <= w_lo && j0 > w_hi - window;
      u32x4 pf[2][2];
#pragma unroll
      for (int a = 0; a < 2; ++a) {
        const int qi = w_lo + a * 16 + n;
        float mx = m[a];
#pragma unroll
        for (int t = 0; t < 4; ++t) s[a][t] *= scale_log2;
        if (!whole) {
          const int age = qi - j0 - g * 4;  // of key (t, i): age - 16t - i
#pragma unroll
          for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int i = 0; i < 4; ++i)
              s[a][t][i] = (unsigned)(age - t * 16 - i) < (unsigned)window
                               ? s[a][t][i]
                               : -INFINITY;
        }
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
          pf[a][p] = u32x4{pack2(s[a][2 * p][0], s[a][2 * p][1]),
                           pack2(s[a][2 * p][2], s[a][2 * p][3]),
                           pack2(s[a][2 * p + 1][0], s[a][2 * p + 1][1]),
                           pack2(s[a][2 * p + 1][2], s[a][2 * p + 1][3])};
      }
#pragma unroll
      for (int v = 0; v < VT; ++v)
#pragma unroll
        for (int p = 0; p < 2; ++p) {
          const unsigned short* r = &lv[(v * 16 + n) * VP + p * 32 + g * 4];
          const uint2 x = *reinterpret_cast<const uint2*>(r);
          const uint2 y = *reinterpret_cast<const uint2*>(r + 16);
          const u32x4 vf = {x.x, x.y, y.x, y.y};
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
    const float inv = 1.f / sum;
    const int r = wave * 32 + a * 16 + n;
    if (r >= n_q) continue;
    bf16_t* dst = out + ((size_t)(q_row + r) * H + h) * V;
    if (g_off >= 0) {
      const bf16_t* gate =
          proj + (size_t)(q_row + r) * ld + g_off + (size_t)h * V;
#pragma unroll
      for (int v = 0; v < VT; ++v) {
        const int d = v * 16 + g * 4;
        float z[4] = {0.f, 0.f, 0.f, 0.f};
        if ((V & 3) == 0 && (g_off & 3) == 0) {
          if (d < V) load4(gate + d, z);
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (d + i < V) z[i] = to_f(gate[d + i]);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) o[a][v][i] /= 1.f + __expf(-z[i]);
      }
    }
#pragma unroll
    for (int v = 0; v < VT; ++v) {
      const int d = v * 16 + g * 4;
      if ((V & 3) == 0) {
        if (d < V)
          *reinterpret_cast<uint2*>(dst + d) =
              make_uint2(pack2(o[a][v][0] * inv, o[a][v][1] * inv),
                         pack2(o[a][v][2] * inv, o[a][v][3] * inv));
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (d + i < V) dst[d + i] = from_f<bf16_t>(o[a][v][i] * inv);
      }
    }
  }
}

// ---------------------------------------------------------------------------
// Absorbed attention of single tokens.  One workgroup: one query, HT
// tiles of 16 heads, one part of its window.  A tile of 64 / HT latents
// goes through LDS; each wave scores 16 of them for one head tile, the
// probabilities go through LDS, and each wave accumulates a quarter of
// the rank for all heads.
//   qa [H][N][rank]; parts: acc [N][H][parts][rank] and (max, sum)
template <int NT, int HT>
__global__ __launch_bounds__(256, NT == 8 && HT == 1 ? 1 : 2)
void latent_decode_kernel(
    bf16_t* __restrict__ out, float* __restrict__ ws_acc,
    float* __restrict__ ws_ml, const bf16_t* __restrict__ qa,
    const bf16_t* __restrict__ proj, int ld, int D, int R, int rank, int H,
    const bf16_t* __restrict__ cache, const int* __restrict__ pos_,
    const int* __restrict__ row_, const int* __restrict__ bt, int max_blocks,
    int window, float scale_log2, const float* __restrict__ sink, int N,
    int parts) {
  constexpr int KD = NT * 2 + 2;         // 32-wide steps over rank + R
  constexpr int KEYS = 64 / HT, KT = KEYS / 16;
  constexpr int PITCH = KD * 32 + 8;
  constexpr int PAGES = KEYS / PAGE;
  constexpr int PL = (PAGE * KD * 4 + 255) / 256;  // loads per page
  constexpr int PP = KEYS + 8;
  extern __shared__ unsigned short lk[];  // KEYS x PITCH
  __shared__ unsigned short lp[HT * 16 * PP];
  __shared__ float lmax[HT * 16][KT], lsum[HT * 16][KT];
  const int q = blockIdx.x, part = blockIdx.z;
  const int h0 = blockIdx.y * HT * 16;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & 63;
  const int n = lane & 15, g = lane >> 4;
  const int kt = wave % KT, ht = wave / KT;  // this wave's scores
  const int width = rank + R, pieces = width / 8;

  const int pos = pos_[q], row = row_[q];
  const int first = pos - window + 1 > 0 ? pos - window + 1 : 0;
  const int base = first & ~(PAGE - 1);  // tiles are whole pages
  const int tiles = (pos - base + KEYS) / KEYS;
  const int per = (tiles + parts - 1) / parts;
  const int t_lo = part * per;
  const int t_hi = t_lo + per < tiles ? t_lo + per : tiles;
  const int* pages = bt + (size_t)row * max_blocks;
  const int last_page = pos / PAGE;

  // the thread's pieces of a page, as offsets into it and into LDS
  // (threads past the last piece repeat it)
  int p_from[PL], p_to[PL], p_row[PL];
#pragma unroll
  for (int i = 0; i < PL; ++i) {
    int p = tid + i * 256;
    p = p < PAGE * pieces ? p : PAGE * pieces - 1;
    p_from[i] = p * 8;
    p_row[i] = p / pieces;
    p_to[i] = p_row[i] * PITCH + p % pieces * 8;
  }
  // page numbers are wave-uniform and fetched a tile ahead of the rows
  int pg[PAGES];
  auto fetch_pages = [&](int t) {
#pragma unroll
    for (int i = 0; i < PAGES; ++i) {
      const int b = base / PAGE + t * PAGES + i;
      pg[i] = pages[b < last_page ? b : last_page];
    }
  };
  u32x4 pk[PAGES][PL];
  auto fetch = [&](int t) {
#pragma unroll
    for (int k = 0; k < PAGES; ++k) {
      const bf16_t* src =
          cache + (size_t)__builtin_amdgcn_readfirstlane(pg[k]) * PAGE * width;
#pragma unroll
      for (int i = 0; i < PL; ++i)
        pk[k][i] = *reinterpret_cast<const u32x4*>(src + p_from[i]);
    }
    if (t + 1 < t_hi) fetch_pages(t + 1);
  };
  if (t_lo < t_hi) fetch_pages(t_lo);
  if (t_lo < t_hi) fetch(t_lo);

  u32x4 qf[KD];
  {
    const int h = h0 + ht * 16 + n;
    const bf16_t* c = qa + ((size_t)(h < H ? h : 0) * N + q) * rank;
    const bf16_t* r = proj + (size_t)q * ld +
                      (size_t)(h < H ? h : 0) * (D + R) + D;
#pragma unroll
    for (int k = 0; k < KD; ++k) {
      const int d = k * 32 + g * 8;
      qf[k] = h >= H || d >= width ? u32x4{0, 0, 0, 0}
              : d < rank ? *reinterpret_cast<const u32x4*>(c + d)
                         : *reinterpret_cast<const u32x4*>(r + (d - rank));
    }
  }
  // columns past the row's end take part in products: keep them zero
  for (int i = tid; i < KEYS * (PITCH / 8); i += 256) {
    const int d = (i % (PITCH / 8)) * 8;
    if (d >= width)
      *reinterpret_cast<u32x4*>(&lk[(i / (PITCH / 8)) * PITCH + d]) =
          u32x4{0, 0, 0, 0};
  }

  f32x4 o[HT][NT];
  float m[HT], l = 0.f;  // m of head n per tile; l of this wave's keys
  // the sink counts once: in the first part, with the first keys
  const bool sunk = sink && part == 0;
  if (sunk && kt == 0 && g == 0) l = 1.f;
#pragma unroll
  for (int a = 0; a < HT; ++a) {
    const int h = h0 + a * 16 + n;
    m[a] = sunk ? sink[h < H ? h : 0] * LOG2E : -1e30f;
#pragma unroll
    for (int t = 0; t < NT; ++t) o[a][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  for (int t = t_lo; t < t_hi; ++t) {
    // rows past the last key meet zero weights and must be finite
    const int left = pos - base - t * KEYS;
    if (left < KEYS - 1) {
#pragma unroll
      for (int k = 0; k < PAGES; ++k)
#pragma unroll
        for (int i = 0; i < PL; ++i)
          if (k * PAGE + p_row[i] > left) pk[k][i] = u32x4{0, 0, 0, 0};
    }
#pragma unroll
    for (int k = 0; k < PAGES; ++k)
#pragma unroll
      for (int i = 0; i < PL; ++i)
        *reinterpret_cast<u32x4*>(&lk[k * PAGE * PITCH + p_to[i]]) =
            pk[k][i];
    __syncthreads();
    if (t + 1 < t_hi) fetch(t + 1);
    f32x4 s = {0.f, 0.f, 0.f, 0.f}, s1 = s;
#pragma unroll
    for (int k = 0; k < KD; k += 2) {
      const unsigned short* c =
          &lk[(kt * 16 + n) * PITCH + k * 32 + g * 8];
      s = mfma(*reinterpret_cast<const u32x4*>(c), qf[k], s);
      s1 = mfma(*reinterpret_cast<const u32x4*>(c + 32), qf[k + 1], s1);
    }
    s += s1;
    const int j = base + t * KEYS + kt * 16 + g * 4;
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      s[i] = j + i >= first && j + i <= pos ? s[i] * scale_log2
                                            : -INFINITY;
      mx = fmaxf(mx, s[i]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
    mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
    if (g == 0) lmax[ht * 16 + n][kt] = mx;
    __syncthreads();
    float keep[HT];
#pragma unroll
    for (int a = 0; a < HT; ++a) {
      float x = m[a];
#pragma unroll
      for (int i = 0; i < KT; ++i) x = fmaxf(x, lmax[a * 16 + n][i]);
      keep[a] = __builtin_amdgcn_exp2f(m[a] - x);
      m[a] = x;
    }
    float mine = m[0], kmine = keep[0];
#pragma unroll
    for (int a = 1; a < HT; ++a)
      if (ht == a) {
        mine = m[a];
        kmine = keep[a];
      }
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      s[i] = __builtin_amdgcn_exp2f(s[i] - mine);
      sum += s[i];
    }
    l = l * kmine + sum;
    *reinterpret_cast<uint2*>(&lp[(ht * 16 + n) * PP + kt * 16 + g * 4]) =
        make_uint2(pack2(s[0], s[1]), pack2(s[2], s[3]));
    __syncthreads();
#pragma unroll
    for (int a = 0; a < HT; ++a)
#pragma unroll
      for (int r = 0; r < NT; ++r) o[a][r] *= keep[a];
#pragma unroll
    for (int ks = 0; ks < KEYS / 32; ++ks) {
      u32x4 pf[HT];
#pragma unroll
      for (int a = 0; a < HT; ++a)
        pf[a] = *reinterpret_cast<const u32x4*>(
            &lp[(a * 16 + n) * PP + ks * 32 + g * 8]);
#pragma unroll
      for (int r = 0; r < NT; ++r) {
        const u32x4 cf = load_columns(
            &lk[(ks * 32 + g * 8 + (n >> 2)) * PITCH +
                (wave * NT + r) * 16 + (n & 3) * 4],
            4 * PITCH);
#pragma unroll
        for (int a = 0; a < HT; ++a) o[a][r] = mfma(cf, pf[a], o[a][r]);
      }
    }
    __syncthreads();
  }
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  if (g == 0) lsum[ht * 16 + n][kt] = l;
  __syncthreads();
#pragma unroll
  for (int a = 0; a < HT; ++a) {
    const int h = h0 + a * 16 + n;
    if (h >= H) continue;
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < KT; ++i) sum += lsum[a * 16 + n][i];
    if (parts == 1) {
      const float inv = 1.f / sum;
      bf16_t* dst = out + ((size_t)h * N + q) * rank;
#pragma unroll
      for (int r = 0; r < NT; ++r) {
        const int d = (wave * NT + r) * 16 + g * 4;
        if (d < rank)  // rank is a multiple of 8
          *reinterpret_cast<uint2*>(dst + d) =
              make_uint2(pack2(o[a][r][0] * inv, o[a][r][1] * inv),
                         pack2(o[a][r][2] * inv, o[a][r][3] * inv));
      }
    } else {
      const size_t at = ((size_t)q * H + h) * parts + part;
#pragma unroll
      for (int r = 0; r < NT; ++r) {
        const int d = (wave * NT + r) * 16 + g * 4;
        if (d < rank)
          *reinterpret_cast<float4*>(ws_acc + at * rank + d) = make_float4(
              o[a][r][0], o[a][r][1], o[a][r][2], o[a][r][3]);
      }
      if (wave == 0 && g == 0) {
        ws_ml[at * 2] = m[a];
        ws_ml[at * 2 + 1] = sum;
      }
    }
  }
}

__global__ __launch_bounds__(256) void latent_merge_kernel(
    bf16_t* __restrict__ out, const float* __restrict__ ws_acc,
    const float* __restrict__ ws_ml, int rank, int H, int N, int parts) {
  const int q = blockIdx.x, h = blockIdx.y;
  const size_t at = ((size_t)q * H + h) * parts;
  float mx = -1e30f;
  for (int p = 0; p < parts; ++p) mx = fmaxf(mx, ws_ml[(at + p) * 2]);
  float sum = 0.f;
  for (int p = 0; p < parts; ++p)
    sum += ws_ml[(at + p) * 2 + 1] *
           __builtin_amdgcn_exp2f(ws_ml[(at + p) * 2] - mx);
  const float inv = 1.f / sum;
  for (int d = threadIdx.x; d < rank; d += 256) {
    float v = 0.f;
    for (int p = 0; p < parts; ++p)
      v += ws_acc[(at + p) * rank + d] *
           __builtin_amdgcn_exp2f(ws_ml[(at + p) * 2] - mx);
    out[((size_t)h * N + q) * rank + d] = from_f<bf16_t>(v * inv);
  }
}

template <int NT, int HT>
static int launch_decode(void* out, void* acc, void* ml, const void* qa,
                         const void* proj, int ld, int D, int R, int rank,
                         int H, const void* cache, const void* pos,
                         const void* row, const void* bt, int max_blocks,
                         int window, float scale, const void* sink, int N,
                         int parts, hipStream_t s) {
  constexpr int lds = (64 / HT) * ((NT * 2 + 2) * 32 + 8) * 2;
  static const hipError_t ready = hipFuncSetAttribute(
      reinterpret_cast<const void*>(latent_decode_kernel<NT, HT>),
      hipFuncAttributeMaxDynamicSharedMemorySize, lds);
  if (ready != hipSuccess) return -3;
  const dim3 grid(N, (H + 16 * HT - 1) / (16 * HT), parts), block(256);
  hipLaunchKernelGGL((latent_decode_kernel<NT, HT>), grid, block, lds, s,
                     (bf16_t*)out, (float*)acc, (float*)ml,
                     (const bf16_t*)qa, (const bf16_t*)proj, ld, D, R, rank,
                     H, (const bf16_t*)cache, (const int*)pos,
                     (const int*)row, (const int*)bt, max_blocks, window,
                     scale * LOG2E, (const float*)sink, N, parts);
  HY_CHECK();
  if (parts > 1) {
    hipLaunchKernelGGL(latent_merge_kernel, dim3(N, H), block, 0, s,
                       (bf16_t*)out, (const float*)acc, (const float*)ml,
                       rank, H, N, parts);
    HY_CHECK();
  }
  return 0;
}

extern "C" {

int hy_latent_gather(void* c, void* kr, const void* cache, const void* blocks,
                     int n_blocks, const void* bt, int max_blocks, int rank,
                     int R, void* stream) {
  if (rank % 8 || R % 8) return -2;
  if (n_blocks <= 0) return 0;
  hipLaunchKernelGGL(latent_gather_kernel, dim3(n_blocks * 4), dim3(256), 0,
                     (hipStream_t)stream, (bf16_t*)c, (bf16_t*)kr,
                     (const bf16_t*)cache, (const int*)blocks,
                     (const int*)bt, max_blocks, rank, R);
  HY_CHECK();
  return 0;
}

int hy_latent_flash(void* out, const void* proj, int ld, const void* kx,
                    const void* kr, const void* vt, int key_ld,
                    const void* items, int n_items, int H, int D, int R,
                    int V, int window, float scale, const void* sink,
                    int g_off, void* stream) {
  if (D % 8 || R % 8 || ld % 8 || key_ld % 64 || D + R > 256 || V > 256)
    return -2;
  if (n_items <= 0) return 0;
  const dim3 grid((unsigned)n_items * H), block(256);
#define GO(DQ, DV)                                                          \
  hipLaunchKernelGGL((latent_flash_kernel<DQ, DV>), grid, block, 0,         \
                     (hipStream_t)stream, (bf16_t*)out,                     \
                     (const bf16_t*)proj, ld, (const bf16_t*)kx,            \
                     (const bf16_t*)kr, (const bf16_t*)vt, key_ld,          \
                     (const int*)items, H, D, R, V, window, scale * LOG2E,  \
                     (const float*)sink, g_off)
  const int dq = D + R;
  if (V <= 64) {
    if (dq <= 64) GO(64, 64);
    else if (dq <= 96) GO(96, 64);
    else if (dq <= 128) GO(128, 64);
    else if (dq <= 192) GO(192, 64);
    else GO(256, 64);
  } else if (V <= 128) {
    if (dq <= 96) GO(96, 128);
    else if (dq <= 128) GO(128, 128);
    else if (dq <= 192) GO(192, 128);
    else GO(256, 128);
  } else {
    GO(256, 256);
  }
#undef GO
  HY_CHECK();
  return 0;
}

int hy_latent_decode(void* out, void* acc, void* ml, const void* qa,
                     const void* proj, int ld, int H, int D, int R, int rank,
                     const void* cache, const void* pos, const void* row,
                     const void* bt, int max_blocks, int window, float scale,
                     const void* sink, int N, int parts, void* stream) {
  if (rank % 8 || R % 8 || D % 8 || ld % 8 || R > 64 || rank > 512 ||
      window <= 0 || parts < 1 || parts > 65535)
    return -2;
  if (N <= 0) return 0;
#define GO(NT)                                                               \
  return H <= 16                                                             \
             ? launch_decode<NT, 1>(out, acc, ml, qa, proj, ld, D, R, rank,  \
                                    H, cache, pos, row, bt, max_blocks,      \
                                    window, scale, sink, N, parts,           \
                                    (hipStream_t)stream)                     \
             : launch_decode<NT, 2>(out, acc, ml, qa, proj, ld, D, R, rank,  \
                                    H, cache, pos, row, bt, max_blocks,      \
                                    window, scale, sink, N, parts,           \
                                    (hipStream_t)stream)
  if (rank <= 64) GO(1);
  if (rank <= 128) GO(2);
  if (rank <= 256) GO(4);
  GO(8);
#undef GO
}

}  // extern "C"
