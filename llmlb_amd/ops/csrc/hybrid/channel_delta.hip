// Gated delta rule with one decay per head and key channel.
//
// Per head, with S [D key channels x V value channels] in float:
//   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// q and k are unit vectors (q times D^-1/2); q, k and v pass a short
// causal convolution and silu first.
//
// Tokens of several sequences lie packed one after another.  Per token:
// pos (place in its sequence), row (its state slot), tstart / tend (its
// sequence's first packed token and the one after its last).
//
// State of a layer
//   S     [slots][H][V][D] float: value-major, so that 16 neighbouring
//         lanes hold one value column and read it in one run
//   ring  [slots][taps][C]: the convolution's last inputs, position p in
//         entry p % taps, C = 2 KH D + H V channels (q, k, v).  The entry
//         of the current token is never one that its own taps read, so
//         decode workgroups of different heads may update it in any order.
// A sequence at position 0 starts from zero whatever its slot holds.
//
// A column of S never meets another, so the prefill scan gives each wave
// 4 columns and walks its sequence's tokens alone: the decayed state is
// multiplied with k AND q in one pass and
//   o = S'^T q + (k . q) u,   S' = diag(g) S
// leaves one cross-lane sum on the critical path of a token.
#include "recurrent.h"

__device__ __forceinline__ float decay_of(float z, float a_log) {
  return expf(-expf(a_log) * softplus_f(z));
}

// Everything that enters the recurrence, in float.  One wave per unit:
// units [0, KH) a q/k head, units [KH, KH + H) a value head.
// ws layout per token: q [KH D] | k [KH D] | g [H D] | v [H V] |
// qk [KH] | beta [H], padded to whole 16-byte vectors.
struct WsLayout {
  int g, v, qk, beta, size;
  __host__ __device__ WsLayout(int KH, int H, int D, int V)
      : g(2 * KH * D), v(g + H * D), qk(v + H * V), beta(qk + KH),
        size((beta + H + 3) & ~3) {}
};

template <typename T, int NJ>
__global__ __launch_bounds__(256) void delta_prep_kernel(
    float* __restrict__ ws, const T* __restrict__ proj, int ld, int b_off,
    const T* __restrict__ dec, const T* __restrict__ ring,
    const float* __restrict__ wconv, const float* __restrict__ a_log,
    const float* __restrict__ dt_bias, const int* __restrict__ pos_,
    const int* __restrict__ row_, const int* __restrict__ tstart_, int KH,
    int H, int D, int V, int taps, float q_scale) {
  const int t = blockIdx.x;
  const int unit = blockIdx.y * 4 + threadIdx.x / WAVE;
  if (unit >= KH + H) return;
  const int lane = threadIdx.x & (WAVE - 1);
  const int pos = pos_[t], slot = row_[t], ts = tstart_[t];
  const int C = 2 * KH * D + H * V;
  const WsLayout at(KH, H, D, V);
  float* w = ws + (size_t)t * at.size;
  if (unit < KH) {
    float q[NJ], k[NJ], qq = 0.f, kk = 0.f, qk = 0.f;
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      const int d = lane + j * WAVE;
      q[j] = k[j] = 0.f;
      if (d < D) {
        q[j] = conv_silu(proj, ld, ring, wconv, nullptr, C, taps, unit * D + d, t,
                         pos, ts, slot);
        k[j] = conv_silu(proj, ld, ring, wconv, nullptr, C, taps,
                         (KH + unit) * D + d, t, pos, ts, slot);
      }
      qq += q[j] * q[j];
      kk += k[j] * k[j];
    }
    const float qs = q_scale / sqrtf(wave_sum(qq) + 1e-6f);
    const float ks = 1.f / sqrtf(wave_sum(kk) + 1e-6f);
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      const int d = lane + j * WAVE;
      q[j] *= qs;
      k[j] *= ks;
      qk += q[j] * k[j];
      if (d < D) {
        w[unit * D + d] = q[j];
        w[(KH + unit) * D + d] = k[j];
      }
    }
    qk = wave_sum(qk);
    if (lane == 0) w[at.qk + unit] = qk;
  } else {
    const int h = unit - KH;
    for (int j = lane; j < V; j += WAVE) {
      const int c = 2 * KH * D + h * V + j;
      w[at.v + h * V + j] =
          conv_silu(proj, ld, ring, wconv, nullptr, C, taps, c, t, pos, ts, slot);
    }
    const float a = a_log[h];
    for (int d = lane; d < D; d += WAVE)
      w[at.g + h * D + d] = decay_of(
          to_f(dec[(size_t)t * H * D + h * D + d]) + dt_bias[h * D + d], a);
    if (lane == 0)
      w[at.beta + h] =
          sigmoid_f(to_f(proj[(size_t)t * ld + b_off + h]));
  }
}

// delta_prep for at most TAPS_MAX taps and D <= 256: a workgroup walks
// PREP_TOK tokens.  blockIdx.y ranges: q/k heads (16 lanes a head, 16
// heads a workgroup), then value channels, then decays (8 channels a
// thread).  VEC: all sections start on whole vectors.
#define PREP_TOK 16
template <typename T, int RPL, bool VEC>
__global__ __launch_bounds__(256) void delta_prep_run_kernel(
    float* __restrict__ ws, const T* __restrict__ proj, int ld, int b_off,
    const T* __restrict__ dec, const T* __restrict__ ring,
    const float* __restrict__ wconv, const float* __restrict__ a_log,
    const float* __restrict__ dt_bias, const int* __restrict__ pos_,
    const int* __restrict__ row_, const int* __restrict__ tstart_, int n_tok,
    int KH, int H, int D, int V, int taps, float q_scale, int qk_blocks,
    int v_blocks) {
  const int t0 = blockIdx.x * PREP_TOK;
  const int t1 = t0 + PREP_TOK < n_tok ? t0 + PREP_TOK : n_tok;
  const int C = 2 * KH * D + H * V;
  const WsLayout at(KH, H, D, V);
  int y = blockIdx.y;
  if (y < qk_blocks) {
    const int unit = y * 16 + threadIdx.x / 16;
    if (unit >= KH) return;  // whole groups of 16 lanes
    const int r0 = (threadIdx.x & 15) * RPL;
    const int valid = D - r0 < RPL ? (D - r0 > 0 ? D - r0 : 0) : RPL;
    const int cq = unit * D + (valid ? r0 : 0), ck = KH * D + cq;
    ConvRun<T, RPL, VEC> q(proj, ld, ring, wconv, nullptr, C, taps, cq,
                           valid);
    ConvRun<T, RPL, VEC> k(proj, ld, ring, wconv, nullptr, C, taps, ck,
                           valid);
    for (int t = t0; t < t1; ++t) {
      const int ts = tstart_[t];
      if (t == t0 || t == ts) {
        q.start(t, pos_[t], ts, row_[t]);
        k.start(t, pos_[t], ts, row_[t]);
      }
      float a[RPL], b[RPL], qq = 0.f, kk = 0.f, qk = 0.f;
      q.step(t, a);
      k.step(t, b);
#pragma unroll
      for (int i = 0; i < RPL; ++i) {
        if (!VEC && i >= valid) a[i] = b[i] = 0.f;
        qq += a[i] * a[i];
        kk += b[i] * b[i];
        qk += a[i] * b[i];
      }
      const float qs = q_scale / sqrtf(row16_sum(qq) + 1e-6f);
      const float ks = 1.f / sqrtf(row16_sum(kk) + 1e-6f);
      qk = row16_sum(qk) * qs * ks;
#pragma unroll
      for (int i = 0; i < RPL; ++i) {
        a[i] *= qs;
        b[i] *= ks;
      }
      float* w = ws + (size_t)t * at.size;
      store_some<RPL, VEC>(w + cq, valid, a);
      store_some<RPL, VEC>(w + ck, valid, b);
      if ((threadIdx.x & 15) == 0) w[at.qk + unit] = qk;
    }
    return;
  }
  y -= qk_blocks;
  if (y < v_blocks) {
    const int j = (y * 256 + threadIdx.x) * 8;
    if (j >= H * V) return;
    const int valid = H * V - j < 8 ? H * V - j : 8;
    ConvRun<T, 8, VEC> v(proj, ld, ring, wconv, nullptr, C, taps,
                         2 * KH * D + j, valid);
    for (int t = t0; t < t1; ++t) {
      const int ts = tstart_[t];
      if (t == t0 || t == ts) v.start(t, pos_[t], ts, row_[t]);
      float f[8];
      v.step(t, f);
      store_some<8, VEC>(ws + (size_t)t * at.size + at.v + j, valid, f);
    }
    return;
  }
  y -= v_blocks;
  const int j = (y * 256 + threadIdx.x) * 8;
  if (y == 0)
    for (int i = threadIdx.x; i < (t1 - t0) * H; i += 256) {
      const int t = t0 + i / H, h = i % H;
      ws[(size_t)t * at.size + at.beta + h] =
          sigmoid_t<T>(to_f(proj[(size_t)t * ld + b_off + h]));
    }
  if (j >= H * D) return;
  const int valid = H * D - j < 8 ? H * D - j : 8;
  float bias[8], rate[8];
  load_some<8, VEC>(dt_bias + j, valid, bias);
#pragma unroll
  for (int i = 0; i < 8; ++i)
    rate[i] = i < valid ? expf(a_log[(j + i) / D]) : 0.f;
  for (int t = t0; t < t1; ++t) {
    float f[8];
    load_some<8, VEC>(dec + (size_t)t * H * D + j, valid, f);
#pragma unroll
    for (int i = 0; i < 8; ++i) f[i] = decay_t<T>(f[i] + bias[i], rate[i]);
    store_some<8, VEC>(ws + (size_t)t * at.size + at.g + j, valid, f);
  }
}

// One wave = 4 CPL value columns of one head of one sequence: 16 lanes a
// column, RPL key channels and CPL columns a lane.  The operands of the
// next PF tokens are in flight while a token is worked on; they are the
// same for every column, so CPL > 1 divides the load on the vector
// memory path, which is what limits a chip full of waves.
template <int RPL, bool EXACT, int CPL>
__global__ __launch_bounds__(64) void delta_scan_kernel(
    float* __restrict__ o, float* __restrict__ state,
    const float* __restrict__ ws, const int* __restrict__ e_start,
    const int* __restrict__ e_len, const int* __restrict__ e_pos,
    const int* __restrict__ e_row, int KH, int H, int D, int V) {
  constexpr int PF = RPL <= 8 ? 4 : (RPL == 16 ? 2 : 1);
  const int e = blockIdx.y;
  const int nb = (V + 4 * CPL - 1) / (4 * CPL);
  int head, cb;
  if (H % 8 == 0) {  // all columns of a head on one XCD: its L2 serves them
    const int x = blockIdx.x & 7, r = blockIdx.x >> 3;
    head = x * (H / 8) + r / nb;
    cb = r % nb;
  } else {
    head = blockIdx.x / nb;
    cb = blockIdx.x % nb;
  }
  const int lane = threadIdx.x;
  const int col = (cb * 4 + lane / 16) * CPL;  // the lane's first column
  const int r0 = (lane & 15) * RPL;
  const int kh = head / (H / KH);
  const WsLayout at(KH, H, D, V);
  const int len = e_len[e];
  const float* base = ws + (size_t)e_start[e] * at.size;
  float* out = o + ((size_t)e_start[e] * H + head) * V;
  float* sp = state + ((size_t)e_row[e] * H + head) * V * D;
  int cc[CPL];
#pragma unroll
  for (int c = 0; c < CPL; ++c) cc[c] = col + c < V ? col + c : V - 1;

  float S[CPL][RPL];
  const bool resume = e_pos[e] > 0;
#pragma unroll
  for (int c = 0; c < CPL; ++c) {
#pragma unroll
    for (int i = 0; i < RPL; ++i) S[c][i] = 0.f;
    if (resume) load_rows<RPL, EXACT>(sp + (size_t)cc[c] * D, r0, D, S[c]);
  }

  float q[PF][RPL], k[PF][RPL], g[PF][RPL], v[PF][CPL], qk[PF], beta[PF];
  auto fetch = [&](int s, int t) {
    const float* w = base + (size_t)(t < len ? t : len - 1) * at.size;
    load_rows<RPL, EXACT>(w + (size_t)kh * D, r0, D, q[s]);
    load_rows<RPL, EXACT>(w + (size_t)(KH + kh) * D, r0, D, k[s]);
    load_rows<RPL, EXACT>(w + at.g + (size_t)head * D, r0, D, g[s]);
#pragma unroll
    for (int c = 0; c < CPL; ++c) v[s][c] = w[at.v + head * V + cc[c]];
    qk[s] = w[at.qk + kh];
    beta[s] = w[at.beta + head];
  };
#pragma unroll
  for (int s = 0; s < PF; ++s) fetch(s, s);

  // Every lane stores, the same value from several of them (and columns
  // past the last one repeat it): no branch between the loads in flight
  // and their use, so that waiting for one token's operands does not
  // wait for the next ones'.
  int oc = cc[0];
#pragma unroll
  for (int c = 1; c < CPL; ++c) oc = lane % CPL == c ? cc[c] : oc;
  auto token = [&](int s, int t) {
    float a[CPL], b[CPL];
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      a[c] = b[c] = 0.f;
#pragma unroll
      for (int i = 0; i < RPL; ++i) {
        S[c][i] *= g[s][i];
        a[c] += k[s][i] * S[c][i];
        b[c] += q[s][i] * S[c][i];
      }
    }
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      a[c] = row16_sum(a[c]);
      b[c] = row16_sum(b[c]);
    }
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      const float u = beta[s] * (v[s][c] - a[c]);
#pragma unroll
      for (int i = 0; i < RPL; ++i) S[c][i] += k[s][i] * u;
      b[c] += qk[s] * u;
    }
    float mine = b[0];
#pragma unroll
    for (int c = 1; c < CPL; ++c) mine = lane % CPL == c ? b[c] : mine;
    out[(size_t)t * H * V + oc] = mine;
  };
  int t0 = 0;
  for (; t0 + PF <= len; t0 += PF) {
#pragma unroll
    for (int s = 0; s < PF; ++s) {
      token(s, t0 + s);
      fetch(s, t0 + s + PF);
    }
  }
#pragma unroll
  for (int s = 0; s < PF; ++s)
    if (t0 + s < len) token(s, t0 + s);
#pragma unroll
  for (int c = 0; c < CPL; ++c)
    if (col + c < V)
      store_rows<RPL, EXACT>(sp + (size_t)(col + c) * D, r0, D, S[c]);
}

// out = o / rms(o) * w * sigmoid(gate) per head; and, once nothing reads
// it any more, the convolution's ring takes the last tokens' inputs.
template <typename T>
__global__ __launch_bounds__(256) void delta_out_kernel(
    T* __restrict__ out, const float* __restrict__ o,
    const T* __restrict__ gate, const float* __restrict__ w, float eps,
    const T* __restrict__ proj, int ld, T* __restrict__ ring,
    const int* __restrict__ pos_, const int* __restrict__ row_,
    const int* __restrict__ tend_, int H, int V, int C, int taps) {
  const int t = blockIdx.x;
  const int h = blockIdx.y * 4 + threadIdx.x / WAVE;
  const int lane = threadIdx.x & (WAVE - 1);
  if (blockIdx.y == 0 && tend_[t] - t <= taps) {
    T* dst = ring + ((size_t)row_[t] * taps + pos_[t] % taps) * C;
    for (int c = threadIdx.x; c < C; c += 256)
      dst[c] = proj[(size_t)t * ld + c];
  }
  if (h >= H) return;
  const size_t base = ((size_t)t * H + h) * V;
  float ssq = 0.f;
  for (int j = lane; j < V; j += WAVE) ssq += o[base + j] * o[base + j];
  const float r = 1.f / sqrtf(wave_sum(ssq) / V + eps);
  for (int j = lane; j < V; j += WAVE)
    out[base + j] =
        from_f<T>(o[base + j] * r * w[j] * sigmoid_f(to_f(gate[base + j])));
}

// The same with 16 lanes a head and RPL value channels a lane (V <= 256);
// VEC: V = 16 RPL.
template <typename T, int RPL, bool VEC>
__global__ __launch_bounds__(256) void delta_out_run_kernel(
    T* __restrict__ out, const float* __restrict__ o,
    const T* __restrict__ gate, const float* __restrict__ w, float eps,
    const T* __restrict__ proj, int ld, T* __restrict__ ring,
    const int* __restrict__ pos_, const int* __restrict__ row_,
    const int* __restrict__ tend_, int H, int V, int C, int taps) {
  const int t = blockIdx.x;
  const int h = blockIdx.y * 16 + threadIdx.x / 16;
  if (blockIdx.y == 0 && tend_[t] - t <= taps) {
    T* dst = ring + ((size_t)row_[t] * taps + pos_[t] % taps) * C;
    for (int c = threadIdx.x; c < C; c += 256)
      dst[c] = proj[(size_t)t * ld + c];
  }
  if (h >= H) return;  // whole groups of 16 lanes
  const int r0 = (threadIdx.x & 15) * RPL;
  const int valid = V - r0 < RPL ? (V - r0 > 0 ? V - r0 : 0) : RPL;
  const size_t at = ((size_t)t * H + h) * V + (valid ? r0 : 0);
  float x[RPL], gt[RPL], wn[RPL], ssq = 0.f;
  load_some<RPL, VEC>(o + at, valid, x);
  load_some<RPL, VEC>(gate + at, valid, gt);
  load_some<RPL, VEC>(w + (valid ? r0 : 0), valid, wn);
#pragma unroll
  for (int i = 0; i < RPL; ++i) ssq += x[i] * x[i];
  const float r = 1.f / sqrtf(row16_sum(ssq) / V + eps);
#pragma unroll
  for (int i = 0; i < RPL; ++i) x[i] *= r * wn[i] * sigmoid_t<T>(gt[i]);
  store_some<RPL, VEC>(out + at, valid, x);
}

// Decode: one token of every sequence, all of the above in one launch.
// One workgroup per (head, sequence); the state's loads are issued
// before the convolution and norms so that these hide behind them.
template <typename T, int RPL, bool EXACT>
__global__ __launch_bounds__(256) void delta_step_kernel(
    T* __restrict__ out, float* __restrict__ state, T* __restrict__ ring,
    const T* __restrict__ proj, int ld, int b_off,
    const T* __restrict__ dec, const T* __restrict__ gate,
    const float* __restrict__ wconv, const float* __restrict__ a_log,
    const float* __restrict__ dt_bias, const float* __restrict__ w_norm,
    const int* __restrict__ pos_, const int* __restrict__ row_, int KH, int H,
    int D, int V, int taps, float q_scale, float eps) {
  constexpr int NU = 64 / RPL > 8 ? 8 : 64 / RPL;  // columns in flight
  constexpr int DP = 16 * RPL;
  extern __shared__ float lds[];
  float* lq = lds;
  float* lk = lq + DP;
  float* lg = lk + DP;
  float* lv = lg + DP;
  float* lo = lv + V;
  __shared__ float red[4][4];
  const int h = blockIdx.x, s = blockIdx.y;
  const int kh = h / (H / KH);
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & (WAVE - 1);
  const int pos = pos_[s], slot = row_[s];
  const int C = 2 * KH * D + H * V;
  const int r0 = (lane & 15) * RPL;
  const int col0 = wave * 4 + lane / 16;
  float* sp = state + ((size_t)slot * H + h) * (size_t)V * D;

  float S[NU][RPL];
  auto fetch = [&](int base) {
#pragma unroll
    for (int n = 0; n < NU; ++n) {
      const int col = base + n * 16 + col0;
      if (pos > 0 && col < V) {
        load_rows<RPL, EXACT>(sp + (size_t)col * D, r0, D, S[n]);
      } else {
#pragma unroll
        for (int i = 0; i < RPL; ++i) S[n][i] = 0.f;
      }
    }
  };
  fetch(0);

  T* keep = ring + ((size_t)slot * taps + pos % taps) * C;
  auto conv = [&](int c) {
    const float y = conv_silu(proj, ld, ring, wconv, nullptr, C, taps, c, s, pos, s,
                              slot);
    keep[c] = proj[(size_t)s * ld + c];
    return y;
  };
  float qq = 0.f, kk = 0.f, qk = 0.f;
  const float a = a_log[h];
  for (int d = tid; d < DP; d += 256) {
    float q = 0.f, k = 0.f, g = 0.f;
    if (d < D) {
      q = conv(kh * D + d);
      k = conv((KH + kh) * D + d);
      g = decay_of(
          to_f(dec[(size_t)s * H * D + h * D + d]) + dt_bias[h * D + d], a);
    }
    lq[d] = q;
    lk[d] = k;
    lg[d] = g;
    qq += q * q;
    kk += k * k;
    qk += q * k;
  }
  for (int j = tid; j < V; j += 256) lv[j] = conv(2 * KH * D + h * V + j);
  qq = wave_sum(qq);
  kk = wave_sum(kk);
  qk = wave_sum(qk);
  if (lane == 0) {
    red[0][wave] = qq;
    red[1][wave] = kk;
    red[2][wave] = qk;
  }
  __syncthreads();
  qq = red[0][0] + red[0][1] + red[0][2] + red[0][3];
  kk = red[1][0] + red[1][1] + red[1][2] + red[1][3];
  qk = red[2][0] + red[2][1] + red[2][2] + red[2][3];
  const float qs = q_scale / sqrtf(qq + 1e-6f);
  const float ks = 1.f / sqrtf(kk + 1e-6f);
  qk *= qs * ks;
  const float beta = sigmoid_f(to_f(proj[(size_t)s * ld + b_off + h]));
  float q[RPL], k[RPL], g[RPL];
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    q[i] = lq[r0 + i] * qs;
    k[i] = lk[r0 + i] * ks;
    g[i] = lg[r0 + i];
  }
  float ssq = 0.f;
  for (int base = 0; base < V; base += NU * 16) {
    if (base) fetch(base);
#pragma unroll
    for (int n = 0; n < NU; ++n) {
      const int col = base + n * 16 + col0;
      float x = 0.f, y = 0.f;
#pragma unroll
      for (int i = 0; i < RPL; ++i) {
        S[n][i] *= g[i];
        x += k[i] * S[n][i];
        y += q[i] * S[n][i];
      }
      x = row16_sum(x);
      y = row16_sum(y);
      if (col < V) {
        const float u = beta * (lv[col] - x);
#pragma unroll
        for (int i = 0; i < RPL; ++i) S[n][i] += k[i] * u;
        store_rows<RPL, EXACT>(sp + (size_t)col * D, r0, D, S[n]);
        const float r = y + qk * u;
        if ((lane & 15) == 0) {
          lo[col] = r;
          ssq += r * r;
        }
      }
    }
  }
  ssq = wave_sum(ssq);
  if (lane == 0) red[3][wave] = ssq;
  __syncthreads();
  ssq = red[3][0] + red[3][1] + red[3][2] + red[3][3];
  const float rn = 1.f / sqrtf(ssq / V + eps);
  const size_t ob = ((size_t)s * H + h) * V;
  for (int j = tid; j < V; j += 256)
    out[ob + j] =
        from_f<T>(lo[j] * rn * w_norm[j] * sigmoid_f(to_f(gate[ob + j])));
}

// every size the kernels of this file can take
static bool delta_ok(int KH, int H, int D, int V, int taps) {
  return KH > 0 && H > 0 && H % KH == 0 && D > 0 && D <= 512 && V > 0 &&
         V <= 4096 && taps > 0;
}

extern "C" {

// floats per token of the workspace between prep and scan
long long hy_delta_ws_floats(int KH, int H, int D, int V) {
  return WsLayout(KH, H, D, V).size;
}

int hy_delta_prep(void* ws, const void* proj, int ld, int b_off,
                  const void* dec, const void* ring, const void* wconv,
                  const void* a_log, const void* dt_bias, const void* pos,
                  const void* row, const void* tstart, int n_tok, int KH,
                  int H, int D, int V, int taps, float q_scale, int dtype,
                  void* stream) {
  if (!delta_ok(KH, H, D, V, taps)) return -2;
  if (n_tok <= 0) return 0;
  if (taps <= TAPS_MAX && D <= 256) {
    const int qk_blocks = (KH + 15) / 16;
    const int v_blocks = (H * V + 2047) / 2048;
    const int g_blocks = (H * D + 2047) / 2048;
    const dim3 grid((n_tok + PREP_TOK - 1) / PREP_TOK,
                    qk_blocks + v_blocks + g_blocks);
    const bool whole = rows_per_lane(D) * 16 == D && D % 8 == 0 &&
                       V % 8 == 0 && ld % 8 == 0;
#define RUN(RPL, VEC)                                                        \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                        \
      (delta_prep_run_kernel<T, RPL, VEC>), grid, dim3(256), 0,              \
      (hipStream_t)stream, (float*)ws, (const T*)proj, ld, b_off,            \
      (const T*)dec, (const T*)ring, (const float*)wconv,                    \
      (const float*)a_log, (const float*)dt_bias, (const int*)pos,           \
      (const int*)row, (const int*)tstart, n_tok, KH, H, D, V, taps,         \
      q_scale, qk_blocks, v_blocks))
#define PICK(RPL)            \
  do {                       \
    if (whole) RUN(RPL, true); \
    else RUN(RPL, false);    \
  } while (0)
    switch (rows_per_lane(D)) {
      case 1: PICK(1); break;
      case 2: PICK(2); break;
      case 4: PICK(4); break;
      case 8: PICK(8); break;
      default: PICK(16); break;
    }
#undef PICK
#undef RUN
    HY_CHECK();
    return 0;
  }
  const dim3 grid(n_tok, (KH + H + 3) / 4), block(256);
#define GO(NJ)                                                               \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                        \
      (delta_prep_kernel<T, NJ>), grid, block, 0, (hipStream_t)stream,       \
      (float*)ws, (const T*)proj, ld, b_off, (const T*)dec, (const T*)ring,  \
      (const float*)wconv, (const float*)a_log, (const float*)dt_bias,       \
      (const int*)pos, (const int*)row, (const int*)tstart, KH, H, D, V,     \
      taps, q_scale))
  if (D <= 64) GO(1);
  else if (D <= 128) GO(2);
  else if (D <= 256) GO(4);
  else GO(8);
#undef GO
  HY_CHECK();
  return 0;
}

int hy_delta_scan(void* o, void* state, const void* ws, const void* e_start,
                  const void* e_len, const void* e_pos, const void* e_row,
                  int n_entries, int KH, int H, int D, int V, void* stream) {
  if (!delta_ok(KH, H, D, V, 1) || n_entries > 65535) return -2;
  if (n_entries <= 0) return 0;
  // wide lanes where they still put waves enough on the 1024 SIMDs
  const long long waves = (long long)n_entries * H * ((V + 3) / 4);
#define GO(CPL)                                                               \
  do {                                                                        \
    const dim3 grid(H * ((V + 4 * CPL - 1) / (4 * CPL)), n_entries);          \
    HY_RPL(D, hipLaunchKernelGGL(                                             \
        (delta_scan_kernel<RPL, EXACT, CPL>), grid, dim3(64), 0,              \
        (hipStream_t)stream, (float*)o, (float*)state, (const float*)ws,      \
        (const int*)e_start, (const int*)e_len, (const int*)e_pos,            \
        (const int*)e_row, KH, H, D, V));                                     \
  } while (0)
  if (V >= 16 && D <= 128 && waves >= 8192) GO(4);
  else if (V >= 8 && D <= 256 && waves >= 2048) GO(2);
  else GO(1);
#undef GO
  HY_CHECK();
  return 0;
}

int hy_delta_out(void* out, const void* o, const void* gate, const void* w,
                 float eps, const void* proj, int ld, void* ring,
                 const void* pos, const void* row, const void* tend,
                 int n_tok, int KH, int H, int D, int V, int taps, int dtype,
                 void* stream) {
  if (!delta_ok(KH, H, D, V, taps)) return -2;
  if (n_tok <= 0) return 0;
  const int C = 2 * KH * D + H * V;
  if (V <= 256) {
    const dim3 grid(n_tok, (H + 15) / 16);
    const bool whole = rows_per_lane(V) * 16 == V;
#define RUN(RPL, VEC)                                                       \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                       \
      (delta_out_run_kernel<T, RPL, VEC>), grid, dim3(256), 0,              \
      (hipStream_t)stream, (T*)out, (const float*)o, (const T*)gate,        \
      (const float*)w, eps, (const T*)proj, ld, (T*)ring, (const int*)pos,  \
      (const int*)row, (const int*)tend, H, V, C, taps))
#define PICK(RPL)            \
  do {                       \
    if (whole) RUN(RPL, true); \
    else RUN(RPL, false);    \
  } while (0)
    switch (rows_per_lane(V)) {
      case 1: PICK(1); break;
      case 2: PICK(2); break;
      case 4: PICK(4); break;
      case 8: PICK(8); break;
      default: PICK(16); break;
    }
#undef PICK
#undef RUN
    HY_CHECK();
    return 0;
  }
  HY_DTYPE(dtype, hipLaunchKernelGGL(
      delta_out_kernel<T>, dim3(n_tok, (H + 3) / 4), dim3(256), 0,
      (hipStream_t)stream, (T*)out, (const float*)o, (const T*)gate,
      (const float*)w, eps, (const T*)proj, ld, (T*)ring, (const int*)pos,
      (const int*)row, (const int*)tend, H, V, C, taps));
  HY_CHECK();
  return 0;
}

int hy_delta_step(void* out, void* state, void* ring, const void* proj,
                  int ld, int b_off, const void* dec, const void* gate,
                  const void* wconv, const void* a_log, const void* dt_bias,
                  const void* w_norm, const void* pos, const void* row,
                  int n_seq, int KH, int H, int D, int V, int taps,
                  float q_scale, float eps, int dtype, void* stream) {
  if (!delta_ok(KH, H, D, V, taps) || n_seq > 65535) return -2;
  if (n_seq <= 0) return 0;
  const size_t lds = (3 * 16 * rows_per_lane(D) + 2 * V) * sizeof(float);
  const dim3 grid(H, n_seq), block(256);
  HY_DTYPE(dtype, HY_RPL(D, hipLaunchKernelGGL(
      (delta_step_kernel<T, RPL, EXACT>), grid, block, lds,
      (hipStream_t)stream, (T*)out, (float*)state, (T*)ring, (const T*)proj,
      ld, b_off, (const T*)dec, (const T*)gate, (const float*)wconv,
      (const float*)a_log, (const float*)dt_bias, (const float*)w_norm,
      (const int*)pos, (const int*)row, KH, H, D, V, taps, q_scale, eps)));
  HY_CHECK();
  return 0;
}

}  // extern "C"
