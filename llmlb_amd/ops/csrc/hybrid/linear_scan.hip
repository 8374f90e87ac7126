// Linear recurrences with a matrix state per head:
//   S <- diag(g) S + k v^T,   o = S^T q,   S [D key channels x V columns]
//
//  * gated linear attention: g per key channel, sigmoid(z)^(1/tau);
//  * Mamba-2: g = exp(-rate dt) per head, v = dt x, and skip x is added to
//    the output; q, k and x come from a short convolution, q and k serve
//    all heads of a group;
//  * matrix memory (mLSTM): g and the weight of v from exponential gates
//    per head, kept in range by a running maximum m; beside S a normaliser
//    n [D], the same recurrence with v = 1, and o is divided by
//    max(|n . q|, exp(-m)) + 1e-6.  n and m are the state's ``extra``:
//    [slots][H][extra_row(D)], n first, m at extra_row(D) - 4.
//
// Tokens of several sequences lie packed one after another.  Per token:
// pos (place in its sequence), row (its state slot), tstart (its
// sequence's first packed token).  A sequence at position 0 starts from
// zero whatever its slot holds.
//
// Everything that enters the state is float; q, k and v keep the storage
// type they were projected or convolved in until they are used.
#include "memory.h"
#include "recurrent.h"

enum Kind { CHANNEL, HEAD, MEMORY };  // gated linear, Mamba-2, mLSTM

// N consecutive elements as they lie in memory, widened on use, so that
// elements in flight take half the registers and nothing waits for them.
// VEC: the address is aligned to the whole run (or to 16 bytes).
template <typename T, int N, bool VEC>
struct Run;
template <int N, bool VEC>
struct Run<float, N, VEC> {
  float f[N];
  __device__ __forceinline__ void load(const float* p, int valid) {
    load_some<N, VEC>(p, valid, f);
  }
  __device__ __forceinline__ void set(int i, float x) { f[i] = x; }
  __device__ __forceinline__ float get(int i) const { return f[i]; }
};
template <int N>
struct Run<bf16_t, N, false> {
  unsigned short u[N];
  __device__ __forceinline__ void load(const bf16_t* p, int valid) {
#pragma unroll
    for (int i = 0; i < N; ++i) u[i] = i < valid ? p[i].u : 0;
  }
  __device__ __forceinline__ void set(int i, bf16_t x) { u[i] = x.u; }
  __device__ __forceinline__ float get(int i) const {
    return __uint_as_float((unsigned)u[i] << 16);
  }
};
template <>
struct Run<bf16_t, 1, true> : Run<bf16_t, 1, false> {};
template <int N>
struct Run<bf16_t, N, true> {
  unsigned w[N / 2];
  __device__ __forceinline__ void load(const bf16_t* p, int) {
    if (N % 8 == 0) {
#pragma unroll
      for (int i = 0; i < N / 8; ++i) {
        const uint4 v = reinterpret_cast<const uint4*>(p)[i];
        w[i * 4] = v.x; w[i * 4 + 1] = v.y;
        w[i * 4 + 2] = v.z; w[i * 4 + 3] = v.w;
      }
    } else if (N == 4) {
      const uint2 v = *reinterpret_cast<const uint2*>(p);
      w[0] = v.x; w[N / 2 - 1] = v.y;
    } else {
      w[0] = *reinterpret_cast<const unsigned*>(p);
    }
  }
  __device__ __forceinline__ float get(int i) const {
    return __uint_as_float(i & 1 ? w[i / 2] & 0xffff0000u : w[i / 2] << 16);
  }
};

// One wave = 4 CPL value columns of one head of one sequence: 16 lanes a
// column, RPL key channels and CPL columns a lane.  The waves of a
// workgroup take neighbouring columns, so that a CU's cache serves them
// the same rows and its SIMDs get the same number of waves.  The operands of the
// next PF tokens are in flight while a token is worked on.  Nothing but
// the state itself carries over from token to token; the sum over lanes
// that makes an output is off that chain.
//   q, k: columns q_off, k_off + group * D; v: v_off + head * V, of rows of
//   ``in``;  g [T][H D] (CHANNEL) or [T][H];  dt [T][H] without CHANNEL
//   skip: [H] (HEAD), exp(-m) [T][H] (MEMORY)
// MEMORY: every wave carries the normaliser as well, from n0 [entries][H][D];
// one of a head's waves leaves the last one in ``extra``.
template <typename T, int RPL, bool VEC, int CPL, Kind KIND>
__global__ __launch_bounds__(256) void linear_scan_kernel(
    float* __restrict__ o, float* __restrict__ state,
    const T* __restrict__ in, int ld, int q_off, int k_off, int v_off,
    const float* __restrict__ g_, const float* __restrict__ dt_,
    const float* __restrict__ skip_, const int* __restrict__ e_start,
    const int* __restrict__ e_len, const int* __restrict__ e_pos,
    const int* __restrict__ e_row, int G, int H, int D, int V,
    float q_scale, const float* __restrict__ n0, float* __restrict__ extra) {
  constexpr bool CHANNEL = KIND == Kind::CHANNEL;
  constexpr bool MEMORY = KIND == Kind::MEMORY;
  constexpr int PF = RPL <= 4 ? 32 / (CPL < 2 ? 2 : CPL)
                              : (RPL == 8 ? 4 : (RPL == 16 ? 2 : 1));
  const int e = blockIdx.y;
  const int waves = blockDim.x / WAVE;
  const int nb = (V + 4 * CPL - 1) / (4 * CPL) / waves;  // whole workgroups
  int head, cb;
  if (H % 8 == 0) {  // all columns of a head on one XCD: its L2 serves them
    const int x = blockIdx.x & 7, r = blockIdx.x >> 3;
    head = x * (H / 8) + r / nb;
    cb = r % nb;
  } else {
    head = blockIdx.x / nb;
    cb = blockIdx.x % nb;
  }
  const int lane = threadIdx.x & (WAVE - 1);
  cb = cb * waves + threadIdx.x / WAVE;
  const int col = (cb * 4 + lane / 16) * CPL;  // the lane's first column
  const int r0 = (lane & 15) * RPL;
  const int valid = D - r0 < RPL ? (D - r0 > 0 ? D - r0 : 0) : RPL;
  const int rr = valid ? r0 : 0;
  const int group = head / (H / G);
  const int len = e_len[e];
  const size_t first = (size_t)e_start[e];
  // a token's rows are the same for the wave, a lane's place in them is
  // a 32-bit offset
  const T* rows = in + first * ld;
  const float* g_rows = g_ + first * H * (CHANNEL ? D : 1);
  const float* dt_rows = CHANNEL ? nullptr : dt_ + first * H;
  const unsigned q_at = (q_off + group * D + rr) * sizeof(T);
  const unsigned k_at = (k_off + group * D + rr) * sizeof(T);
  const unsigned v_at = (v_off + head * V) * sizeof(T);
  const unsigned g_at = (head * D + rr) * sizeof(float);
  // kept in a vector register: scalar loads return out of order, so that
  // waiting for one token's would wait for the next ones' as well
  unsigned head_at = head * sizeof(float);
  asm("" : "+v"(head_at));
  auto place = [](const auto* p, unsigned bytes) {
    return reinterpret_cast<decltype(p)>(
        reinterpret_cast<const char*>(p) + bytes);
  };
  const float skip = KIND == HEAD ? skip_[head] : 0.f;
  const float* e_rows = MEMORY ? skip_ + first * H : nullptr;
  float* out = o + (first * H + head) * V;
  float* sp = state + ((size_t)e_row[e] * H + head) * V * D;
  int cc[CPL];
#pragma unroll
  for (int c = 0; c < CPL; ++c)
    cc[c] = VEC || col + c < V ? col + c : V - 1;

  float S[CPL][RPL], N[RPL];
  if (MEMORY)
    load_rows<RPL, VEC>(n0 + ((size_t)e * H + head) * D, r0, D, N);
  const bool resume = e_pos[e] > 0;
#pragma unroll
  for (int c = 0; c < CPL; ++c) {
#pragma unroll
    for (int i = 0; i < RPL; ++i) S[c][i] = 0.f;
    if (resume) load_rows<RPL, VEC>(sp + (size_t)cc[c] * D, r0, D, S[c]);
  }

  constexpr int GN = CHANNEL ? RPL : 1;
  Run<T, RPL, VEC> q[PF], k[PF];
  Run<T, CPL, VEC> v[PF];
  float g[PF][GN], dt[PF], floor_[MEMORY ? PF : 1];
  auto fetch = [&](int s, int t) {
    t = t < len ? t : len - 1;
    const T* row = rows + (size_t)t * ld;
    q[s].load(place(row, q_at), valid);
    k[s].load(place(row, k_at), valid);
    if (CHANNEL) {
      load_some<GN, VEC>(place(g_rows + (size_t)t * H * D, g_at), valid, g[s]);
      dt[s] = 1.f;
    } else {
      g[s][0] = *place(g_rows + (size_t)t * H, head_at);
      dt[s] = *place(dt_rows + (size_t)t * H, head_at);
      if (MEMORY) floor_[s] = *place(e_rows + (size_t)t * H, head_at);
    }
    if constexpr (VEC) {
      v[s].load(place(row, v_at + col * (unsigned)sizeof(T)), CPL);
    } else {
#pragma unroll
      for (int c = 0; c < CPL; ++c)
        v[s].set(c, *place(row, v_at + cc[c] * (unsigned)sizeof(T)));
    }
  };
#pragma unroll
  for (int s = 0; s < PF; ++s) fetch(s, s);

  // Every lane stores, the same value from several of them (and columns
  // past the last one repeat it): no branch between the loads in flight
  // and their use.
  int oc = cc[0];
#pragma unroll
  for (int c = 1; c < CPL; ++c) oc = lane % CPL == c ? cc[c] : oc;
  auto token = [&](int s, int t) {
    float b[CPL], x[CPL];
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      x[c] = v[s].get(c);
      const float u = x[c] * dt[s];
      b[c] = 0.f;
#pragma unroll
      for (int i = 0; i < RPL; ++i) {
        S[c][i] = S[c][i] * g[s][CHANNEL ? i : 0] + k[s].get(i) * u;
        b[c] += q[s].get(i) * S[c][i];
      }
    }
    float mine;
    if constexpr (CPL == 4) {
      mine = row16_sum4(b);
    } else {
#pragma unroll
      for (int c = 0; c < CPL; ++c) b[c] = row16_sum(b[c]);
      mine = b[0];
#pragma unroll
      for (int c = 1; c < CPL; ++c) mine = lane % CPL == c ? b[c] : mine;
    }
    if (MEMORY) {
      float a = 0.f;
#pragma unroll
      for (int i = 0; i < RPL; ++i) {
        N[i] = N[i] * g[s][0] + k[s].get(i) * dt[s];
        a += q[s].get(i) * N[i];
      }
      a = fabsf(row16_sum(a) * q_scale);
      mine *= q_scale / (fmaxf(a, floor_[MEMORY ? s : 0]) + MEMORY_EPS);
    } else if (!CHANNEL) {
      float xm = x[0];
#pragma unroll
      for (int c = 1; c < CPL; ++c) xm = lane % CPL == c ? x[c] : xm;
      mine += skip * xm;
    } else {
      mine *= q_scale;
    }
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
      store_rows<RPL, VEC>(sp + (size_t)(col + c) * D, r0, D, S[c]);
  if (MEMORY && col == 0)
    store_rows<RPL, VEC>(
        extra + ((size_t)e_row[e] * H + head) * extra_row(D), r0, D, N);
}

// What matrix memory's scan needs of every token and head, one wave per
// (head, entry): the running maximum m as a scan of max(a + ., b), 64
// tokens at a time, then steps [3][T][H] = exp(f + m' - m), exp(i - m),
// exp(-m).  bias [2][H]: input gates', forget gates'.  Also copies the
// normaliser out of the state (several workgroups of the scan read it and
// one replaces it) and leaves the last m there.
template <typename T>
__global__ __launch_bounds__(64) void memory_gates_kernel(
    float* __restrict__ steps, float* __restrict__ n0,
    float* __restrict__ extra, const T* __restrict__ proj, int ld, int i_off,
    int f_off, const float* __restrict__ bias, const int* __restrict__ e_start,
    const int* __restrict__ e_len, const int* __restrict__ e_pos,
    const int* __restrict__ e_row, int n_tok, int H, int D, float cap) {
  const int h = blockIdx.x, e = blockIdx.y, lane = threadIdx.x;
  const int len = e_len[e], first = e_start[e];
  const bool resume = e_pos[e] > 0;
  float* ex = extra + ((size_t)e_row[e] * H + h) * extra_row(D);
  for (int d = lane; d < D; d += WAVE)
    n0[((size_t)e * H + h) * D + d] = resume ? ex[d] : 0.f;
  float m = resume ? ex[extra_row(D) - 4] : 0.f;
  const float bi = bias[h], bf = bias[H + h];
  const size_t plane = (size_t)n_tok * H;
  auto fetch = [&](int t, float& zi, float& zf) {
    t = t < len ? t : len - 1;
    const T* row = proj + (size_t)(first + t) * ld + h;
    zi = to_f(row[i_off]);
    zf = to_f(row[f_off]);
  };
  float zi, zf;
  fetch(lane, zi, zf);
  for (int t0 = 0; t0 < len; t0 += WAVE) {
    const int t = t0 + lane;
    float li, lf;
    memory_gates(zi + bi, zf + bf, cap, li, lf);
    if (t0 + WAVE < len) fetch(t + WAVE, zi, zf);
    float a = lf, b = li;
#pragma unroll
    for (int o = 1; o < WAVE; o <<= 1) {
      const float a1 = __shfl_up(a, o, WAVE), b1 = __shfl_up(b, o, WAVE);
      if (lane >= o) {
        b = fmaxf(b1 + a, b);
        a += a1;
      }
    }
    const float now = fmaxf(a + m, b);
    float before = __shfl_up(now, 1, WAVE);
    if (lane == 0) before = m;
    if (t < len) {
      const size_t at = (size_t)(first + t) * H + h;
      steps[at] = expf(lf + before - now);
      steps[plane + at] = expf(li - now);
      steps[2 * plane + at] = expf(-now);
    }
    const int last = len - t0 < WAVE ? len - t0 - 1 : WAVE - 1;
    m = __shfl(now, last, WAVE);
  }
  if (lane == 0) ex[extra_row(D) - 4] = m;
}

// g = sigmoid(dec + bias)^rate per channel
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void gla_decay_kernel(
    float* __restrict__ g, const T* __restrict__ dec,
    const float* __restrict__ bias, int n_tok, int C, float rate) {
  constexpr int N = VEC ? 8 : 1;
  const int c = (blockIdx.y * 256 + threadIdx.x) * N;
  if (c >= C) return;
  float b[N];
  load_run<N, VEC>(bias + c, b);
  for (int t = blockIdx.x; t < n_tok; t += gridDim.x) {
    float f[N];
    load_run<N, VEC>(dec + (size_t)t * C + c, f);
#pragma unroll
    for (int i = 0; i < N; ++i) f[i] = decay_t<T>(-(f[i] + b[i]), rate);
    store_run<N, VEC>(g + (size_t)t * C + c, f);
  }
}

// dt = softplus(. + bias) and g = exp(-rate dt) of one head and token
__device__ __forceinline__ void ssm_times(float raw, float bias, float rate,
                                          float& dt, float& g) {
  dt = softplus_f(raw + bias);
  g = expf(-rate * dt);
}

// Convolved channels of a packed batch, one channel a thread (any taps).
template <typename T>
__global__ __launch_bounds__(256) void ssm_conv_kernel(
    T* __restrict__ xbc, const T* __restrict__ proj, int ld,
    const T* __restrict__ ring, const float* __restrict__ wconv,
    const float* __restrict__ bias, const int* __restrict__ pos_,
    const int* __restrict__ row_, const int* __restrict__ tstart_, int C,
    int taps) {
  const int t = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  xbc[(size_t)t * C + c] =
      from_f<T>(conv_silu(proj, ld, ring, wconv, bias, C, taps, c, t, pos_[t],
                          tstart_[t], row_[t]));
}

// The same for at most TAPS_MAX taps: 8 channels a thread, each input of
// PREP_TOK successive tokens read once.
#define PREP_TOK 16
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void ssm_conv_run_kernel(
    T* __restrict__ xbc, const T* __restrict__ proj, int ld,
    const T* __restrict__ ring, const float* __restrict__ wconv,
    const float* __restrict__ bias, const int* __restrict__ pos_,
    const int* __restrict__ row_, const int* __restrict__ tstart_, int n_tok,
    int C, int taps) {
  const int t0 = blockIdx.x * PREP_TOK;
  const int t1 = t0 + PREP_TOK < n_tok ? t0 + PREP_TOK : n_tok;
  const int c = (blockIdx.y * 256 + threadIdx.x) * 8;
  if (c >= C) return;
  const int valid = C - c < 8 ? C - c : 8;
  ConvRun<T, 8, VEC> run(proj, ld, ring, wconv, bias, C, taps, c, valid);
  for (int t = t0; t < t1; ++t) {
    const int ts = tstart_[t];
    if (t == t0 || t == ts) run.start(t, pos_[t], ts, row_[t]);
    float f[8];
    run.step(t, f);
    store_some<8, VEC>(xbc + (size_t)t * C + c, valid, f);
  }
}

// steps [2][T][H]: decay and dt.  per_head [3][H]: bias, rate, skip.
template <typename T>
__global__ __launch_bounds__(256) void ssm_times_kernel(
    float* __restrict__ steps, const T* __restrict__ proj, int ld, int dt_off,
    const float* __restrict__ per_head, int n_tok, int H) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= n_tok * H) return;
  const int t = i / H, h = i - t * H;
  float dt, g;
  ssm_times(to_f(proj[(size_t)t * ld + dt_off + h]), per_head[h],
            per_head[H + h], dt, g);
  steps[i] = g;
  steps[n_tok * H + i] = dt;
}

// The last inputs of every entry into its ring, once nothing reads the
// ring any more.
template <typename T>
__global__ __launch_bounds__(256) void ring_store_kernel(
    T* __restrict__ ring, const T* __restrict__ proj, int ld,
    const int* __restrict__ e_start, const int* __restrict__ e_len,
    const int* __restrict__ e_pos, const int* __restrict__ e_row, int C,
    int taps) {
  const int e = blockIdx.x, len = e_len[e];
  const int n = len < taps ? len : taps;
  for (int i = blockIdx.y; i < n; i += gridDim.y) {
    const int j = len - n + i;
    const T* src = proj + (size_t)(e_start[e] + j) * ld;
    T* dst = ring + ((size_t)e_row[e] * taps + (e_pos[e] + j) % taps) * C;
    for (int c = threadIdx.x; c < C; c += 256) dst[c] = src[c];
  }
}

// Decode: one token of every sequence.  One workgroup per (head,
// sequence); the state's loads are issued first so that everything the
// token needs is computed behind them.
//   CHANNEL: gated linear attention, out = silu(gate) norm(o)
//   HEAD: Mamba-2, y = o + skip x (gate and norm span the heads)
//   MEMORY: mLSTM, out = sigmoid(gate) norm(o); ``dec`` points to the
//     input gates' projections (the forget gates' follow), per_head [2][H]
//     are their biases and ``rate`` the cap
template <typename T, int RPL, bool EXACT, Kind KIND>
__global__ __launch_bounds__(256) void linear_step_kernel(
    T* __restrict__ out, int ld_out, float* __restrict__ y,
    float* __restrict__ state, const T* __restrict__ proj, int ld, int q_off,
    int k_off, int v_off, int g_off, const T* __restrict__ dec,
    const float* __restrict__ dec_bias, const float* __restrict__ w_norm,
    T* __restrict__ ring, const float* __restrict__ wconv,
    const float* __restrict__ conv_bias, const float* __restrict__ per_head,
    float* __restrict__ extra, const int* __restrict__ pos_,
    const int* __restrict__ row_, int G, int H, int D, int V, int taps,
    float q_scale, float rate, float eps) {
  constexpr bool CONV = KIND == HEAD;
  constexpr int NU = 64 / RPL > 8 ? 8 : 64 / RPL;  // columns in flight
  constexpr int DP = 16 * RPL;
  extern __shared__ float lds[];
  float* lq = lds;
  float* lk = lq + DP;
  float* lg = lk + DP;
  float* lv = lg + DP;
  float* lo = lv + V;
  __shared__ float red[4];
  const int h = blockIdx.x, s = blockIdx.y;
  const int group = h / (H / G);
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & (WAVE - 1);
  const int pos = pos_[s], slot = row_[s];
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

  const T* row = proj + (size_t)s * ld;
  float gh = 0.f, dt = 1.f, skip = 0.f;
  float N[RPL], m = 0.f, inv = 1.f;
  float* ex = nullptr;
  if constexpr (CONV) {
    const int C = H * V + 2 * G * D;
    T* keep = ring + ((size_t)slot * taps + pos % taps) * C;
    auto conv = [&](int c) {
      const float f = conv_silu(proj, ld, ring, wconv, conv_bias, C, taps, c,
                                s, pos, s, slot);
      keep[c] = row[c];
      return f;
    };
    for (int d = tid; d < DP; d += 256) {
      lq[d] = d < D ? conv(q_off + group * D + d) : 0.f;
      lk[d] = d < D ? conv(k_off + group * D + d) : 0.f;
    }
    for (int j = tid; j < V; j += 256) lv[j] = conv(v_off + h * V + j);
    ssm_times(to_f(row[g_off + h]), per_head[h], per_head[H + h], dt, gh);
    skip = per_head[2 * H + h];
  } else if constexpr (KIND == MEMORY) {
    for (int d = tid; d < DP; d += 256) {
      const bool ok = d < D;
      lq[d] = ok ? to_f(row[q_off + h * D + d]) * q_scale : 0.f;
      lk[d] = ok ? to_f(row[k_off + h * D + d]) : 0.f;
    }
    for (int j = tid; j < V; j += 256) lv[j] = to_f(row[v_off + h * V + j]);
    const T* z = dec + (size_t)s * ld + h;
    float li, lf;
    memory_gates(to_f(z[0]) + per_head[h], to_f(z[H]) + per_head[H + h], rate,
                 li, lf);
    ex = extra + ((size_t)slot * H + h) * extra_row(D);
    const float before = pos > 0 ? ex[extra_row(D) - 4] : 0.f;
    m = fmaxf(lf + before, li);
    gh = expf(lf + before - m);
    dt = expf(li - m);
#pragma unroll
    for (int i = 0; i < RPL; ++i) N[i] = 0.f;
    if (pos > 0) load_rows<RPL, EXACT>(ex, r0, D, N);
  } else {
    for (int d = tid; d < DP; d += 256) {
      const bool ok = d < D;
      lq[d] = ok ? to_f(row[q_off + h * D + d]) * q_scale : 0.f;
      lk[d] = ok ? to_f(row[k_off + h * D + d]) : 0.f;
      lg[d] = ok ? decay_t<T>(-(to_f(dec[((size_t)s * H + h) * D + d]) +
                                dec_bias[h * D + d]),
                              rate)
                 : 0.f;
    }
    for (int j = tid; j < V; j += 256) lv[j] = to_f(row[v_off + h * V + j]);
  }
  __syncthreads();
  float q[RPL], k[RPL], g[RPL];
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    q[i] = lq[r0 + i];
    k[i] = lk[r0 + i] * dt;
    g[i] = KIND == CHANNEL ? lg[r0 + i] : gh;
  }
  if constexpr (KIND == MEMORY) {
    // every 16 lanes make the normaliser; what it was has been read
    float a = 0.f;
#pragma unroll
    for (int i = 0; i < RPL; ++i) {
      N[i] = N[i] * gh + k[i];
      a += q[i] * N[i];
    }
    inv = 1.f / (fmaxf(fabsf(row16_sum(a)), expf(-m)) + MEMORY_EPS);
    if (tid < 16) store_rows<RPL, EXACT>(ex, r0, D, N);
    if (tid == 0) ex[extra_row(D) - 4] = m;
  }
  float ssq = 0.f;
  for (int base = 0; base < V; base += NU * 16) {
    if (base) fetch(base);
#pragma unroll
    for (int n = 0; n < NU; ++n) {
      const int col = base + n * 16 + col0;
      const float v = lv[col < V ? col : 0];
      float r = 0.f;
#pragma unroll
      for (int i = 0; i < RPL; ++i) {
        S[n][i] = S[n][i] * g[i] + k[i] * v;
        r += q[i] * S[n][i];
      }
      r = row16_sum(r);
      if (KIND == MEMORY) r *= inv;
      if (col < V) {
        store_rows<RPL, EXACT>(sp + (size_t)col * D, r0, D, S[n]);
        if ((lane & 15) == 0) {
          lo[col] = r + skip * v;
          ssq += r * r;
        }
      }
    }
  }
  if constexpr (CONV) {
    __syncthreads();
    for (int j = tid; j < V; j += 256)
      y[((size_t)s * H + h) * V + j] = lo[j];
  } else {
    ssq = block_sum_256(ssq, red);
    const float rn = 1.f / sqrtf(ssq / V + eps);
    for (int j = tid; j < V; j += 256) {
      const float z = to_f(row[g_off + h * V + j]);
      const float f = KIND == MEMORY ? w_norm[h * V + j] * sigmoid_f(z)
                                     : w_norm[j] * silu_f(z);
      out[(size_t)s * ld_out + h * V + j] = from_f<T>(lo[j] * rn * f);
    }
  }
}

// every size the kernels of this file can take
static bool scan_ok(int G, int H, int D, int V) {
  return G > 0 && H > 0 && H % G == 0 && D > 0 && D <= 512 && V > 0 &&
         V <= 4096;
}

template <Kind KIND>
static int launch_step(void* out, int ld_out, void* y, void* state,
                       const void* proj, int ld, int q_off, int k_off,
                       int v_off, int g_off, const void* dec,
                       const void* dec_bias, const void* w_norm, void* ring,
                       const void* wconv, const void* conv_bias,
                       const void* per_head, void* extra, const void* pos,
                       const void* row, int n_seq, int G, int H, int D, int V, int taps,
                       float q_scale, float rate, float eps, int dtype,
                       void* stream) {
  if (!scan_ok(G, H, D, V) || n_seq > 65535) return -2;
  if (n_seq <= 0) return 0;
  const size_t lds = (3 * 16 * rows_per_lane(D) + 2 * V) * sizeof(float);
  const dim3 grid(H, n_seq), block(256);
  HY_DTYPE(dtype, HY_RPL(D, hipLaunchKernelGGL(
      (linear_step_kernel<T, RPL, EXACT, KIND>), grid, block, lds,
      (hipStream_t)stream, (T*)out, ld_out, (float*)y, (float*)state,
      (const T*)proj, ld, q_off, k_off, v_off, g_off, (const T*)dec,
      (const float*)dec_bias, (const float*)w_norm, (T*)ring,
      (const float*)wconv, (const float*)conv_bias, (const float*)per_head,
      (float*)extra, (const int*)pos, (const int*)row, G, H, D, V, taps,
      q_scale, rate, eps)));
  HY_CHECK();
  return 0;
}

extern "C" {

int hy_linear_scan(void* o, void* state, const void* in, int ld, int q_off,
                   int k_off, int v_off, const void* g, const void* dt,
                   const void* skip, const void* e_start, const void* e_len,
                   const void* e_pos, const void* e_row, int n_entries, int G,
                   int H, int D, int V, float q_scale, const void* n0,
                   void* extra, int dtype, void* stream) {
  if (!scan_ok(G, H, D, V) || n_entries > 65535) return -2;
  if (n_entries <= 0) return 0;
  const bool channel = dt == nullptr, memory = n0 != nullptr;
  if (channel ? G != H : !skip) return -2;
  if (memory && (channel || !extra)) return -2;
  // wide lanes where they still put waves enough on the 1024 SIMDs
  // (measured; a decay per channel gains more from sharing its loads)
  const long long waves = (long long)n_entries * H * ((V + 3) / 4);
  const bool vec = ld % 8 == 0 && q_off % 8 == 0 && k_off % 8 == 0 &&
                   v_off % 8 == 0 && D % 8 == 0 && V % 16 == 0 &&
                   rows_per_lane(D) * 16 == D;
  // waves of a workgroup: all of a head's column blocks in whole groups
  auto group = [&](int cpl) {
    const int nb = (V + 4 * cpl - 1) / (4 * cpl);
    return nb % 4 == 0 ? 4 : (nb % 2 == 0 ? 2 : 1);
  };
#define RUN(CPL, KIND, VEC)                                                   \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                         \
      (linear_scan_kernel<T, RPL, VEC, CPL, KIND>),                           \
      dim3(H * ((V + 4 * CPL - 1) / (4 * CPL)) / group(CPL), n_entries),      \
      dim3(64 * group(CPL)), 0,                                               \
      (hipStream_t)stream, (float*)o, (float*)state, (const T*)in, ld, q_off, \
      k_off, v_off, (const float*)g, (const float*)dt, (const float*)skip,    \
      (const int*)e_start, (const int*)e_len, (const int*)e_pos,              \
      (const int*)e_row, G, H, D, V, q_scale, (const float*)n0,               \
      (float*)extra))
// (the wide forms are chosen for small D only)
#define PICK(CPL)                               \
  do {                                          \
    if constexpr (RPL * CPL <= 32) {            \
      if (channel && vec) RUN(CPL, CHANNEL, true); \
      else if (channel) RUN(CPL, CHANNEL, false);  \
      else if (memory && vec) RUN(CPL, MEMORY, true); \
      else if (memory) RUN(CPL, MEMORY, false);    \
      else if (vec) RUN(CPL, HEAD, true);          \
      else RUN(CPL, HEAD, false);                  \
    }                                           \
  } while (0)
#define GO(CPL)                                                    \
  do {                                                             \
    switch (rows_per_lane(D)) {                                    \
      case 1: { constexpr int RPL = 1; PICK(CPL); } break;         \
      case 2: { constexpr int RPL = 2; PICK(CPL); } break;         \
      case 4: { constexpr int RPL = 4; PICK(CPL); } break;         \
      case 8: { constexpr int RPL = 8; PICK(CPL); } break;         \
      case 16: { constexpr int RPL = 16; PICK(CPL); } break;       \
      default: { constexpr int RPL = 32; PICK(CPL); } break;       \
    }                                                              \
  } while (0)
  if (V % 16 == 0 && D <= 128 && waves >= (channel ? 4096 : 8192)) GO(4);
  else if (V >= 8 && D <= 256 && waves >= 2048) GO(2);
  else GO(1);
#undef GO
#undef PICK
#undef RUN
  HY_CHECK();
  return 0;
}

int hy_gla_decay(void* g, const void* dec, const void* bias, int n_tok, int C,
                 float rate, int dtype, void* stream) {
  if (n_tok <= 0 || C <= 0) return 0;
  const bool vec = C % 8 == 0;
  const int cols = vec ? 2048 : 256;
  const dim3 grid(n_tok < 2048 ? n_tok : 2048, (C + cols - 1) / cols);
#define GO(VEC)                                                          \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                    \
      (gla_decay_kernel<T, VEC>), grid, dim3(256), 0,                    \
      (hipStream_t)stream, (float*)g, (const T*)dec, (const float*)bias, \
      n_tok, C, rate))
  if (vec) GO(true);
  else GO(false);
#undef GO
  HY_CHECK();
  return 0;
}

int hy_gla_step(void* out, int ld_out, void* state, const void* proj, int ld,
                int k_off, int v_off, int g_off, const void* dec,
                const void* dec_bias, const void* w_norm, const void* pos,
                const void* row, int n_seq, int H, int D, int V,
                float q_scale, float rate, float eps, int dtype,
                void* stream) {
  return launch_step<CHANNEL>(out, ld_out, nullptr, state, proj, ld, 0,
                              k_off, v_off, g_off, dec, dec_bias, w_norm,
                              nullptr, nullptr, nullptr, nullptr, nullptr,
                              pos, row, n_seq, H, H, D, V, 1, q_scale, rate,
                              eps, dtype, stream);
}

int hy_memory_step(void* out, int ld_out, void* state, void* extra,
                   const void* proj, int ld, int k_off, int v_off, int g_off,
                   int i_off, const void* bias, const void* w_norm,
                   const void* pos, const void* row, int n_seq, int H, int D,
                   int V, float q_scale, float cap, float eps, int dtype,
                   void* stream) {
  const size_t esize = dtype == 0 ? 2 : 4;
  return launch_step<MEMORY>(out, ld_out, nullptr, state, proj, ld, 0, k_off,
                             v_off, g_off, (const char*)proj + i_off * esize,
                             nullptr, w_norm, nullptr, nullptr, nullptr, bias,
                             extra, pos, row, n_seq, H, H, D, V, 1, q_scale,
                             cap, eps, dtype, stream);
}

int hy_memory_gates(void* steps, void* n0, void* extra, const void* proj,
                    int ld, int i_off, const void* bias, const void* e_start,
                    const void* e_len, const void* e_pos, const void* e_row,
                    int n_entries, int n_tok, int H, int D, float cap,
                    int dtype, void* stream) {
  if (!scan_ok(H, H, D, 1) || n_entries > 65535 || !(cap > 0.f)) return -2;
  if (n_entries <= 0 || n_tok <= 0) return 0;
  HY_DTYPE(dtype, hipLaunchKernelGGL(
      memory_gates_kernel<T>, dim3(H, n_entries), dim3(WAVE), 0,
      (hipStream_t)stream, (float*)steps, (float*)n0, (float*)extra,
      (const T*)proj, ld, i_off, i_off + H, (const float*)bias,
      (const int*)e_start, (const int*)e_len, (const int*)e_pos,
      (const int*)e_row, n_tok, H, D, cap));
  HY_CHECK();
  return 0;
}

int hy_ssm_step(void* y, void* state, const void* proj, int ld, int dt_off,
                void* ring, const void* wconv, const void* bias,
                const void* per_head, const void* pos, const void* row,
                int n_seq, int G, int H, int N, int V, int taps, int dtype,
                void* stream) {
  if (taps <= 0) return -2;
  return launch_step<HEAD>(nullptr, 0, y, state, proj, ld, H * V + G * N,
                           H * V, 0, dt_off, nullptr, nullptr, nullptr, ring,
                           wconv, bias, per_head, nullptr, pos, row, n_seq, G,
                           H, N, V, taps, 1.f, 0.f, 0.f, dtype, stream);
}

int hy_ssm_prep(void* xbc, void* steps, const void* proj, int ld, int dt_off,
                const void* ring, const void* wconv, const void* bias,
                const void* per_head, const void* pos, const void* row,
                const void* tstart, int n_tok, int C, int H, int taps,
                int dtype, void* stream) {
  if (taps <= 0 || C <= 0 || H <= 0) return -2;
  if (n_tok <= 0) return 0;
  if ((long long)n_tok * H >= (1ll << 30)) return -2;
  hipStream_t st = (hipStream_t)stream;
  if (taps <= TAPS_MAX) {
    const dim3 grid((n_tok + PREP_TOK - 1) / PREP_TOK, (C + 2047) / 2048);
#define GO(VEC)                                                              \
  HY_DTYPE(dtype, hipLaunchKernelGGL(                                        \
      (ssm_conv_run_kernel<T, VEC>), grid, dim3(256), 0, st, (T*)xbc,        \
      (const T*)proj, ld, (const T*)ring, (const float*)wconv,               \
      (const float*)bias, (const int*)pos, (const int*)row,                  \
      (const int*)tstart, n_tok, C, taps))
    if (C % 8 == 0 && ld % 8 == 0) GO(true);
    else GO(false);
#undef GO
  } else {
    HY_DTYPE(dtype, hipLaunchKernelGGL(
        ssm_conv_kernel<T>, dim3(n_tok, (C + 255) / 256), dim3(256), 0, st,
        (T*)xbc, (const T*)proj, ld, (const T*)ring, (const float*)wconv,
        (const float*)bias, (const int*)pos, (const int*)row,
        (const int*)tstart, C, taps));
  }
  HY_CHECK();
  HY_DTYPE(dtype, hipLaunchKernelGGL(
      ssm_times_kernel<T>, dim3((n_tok * H + 255) / 256), dim3(256), 0, st,
      (float*)steps, (const T*)proj, ld, dt_off, (const float*)per_head,
      n_tok, H));
  HY_CHECK();
  return 0;
}

int hy_ring_store(void* ring, const void* proj, int ld, const void* e_start,
                  const void* e_len, const void* e_pos, const void* e_row,
                  int n_entries, int C, int taps, int dtype, void* stream) {
  if (taps <= 0 || C <= 0) return -2;
  if (n_entries <= 0) return 0;
  HY_DTYPE(dtype, hipLaunchKernelGGL(
      ring_store_kernel<T>, dim3(n_entries, taps < 8 ? taps : 8), dim3(256),
      0, (hipStream_t)stream, (T*)ring, (const T*)proj, ld,
      (const int*)e_start, (const int*)e_len, (const int*)e_pos,
      (const int*)e_row, C, taps));
  HY_CHECK();
  return 0;
}

}  // extern "C"
