// What a parallel layer of windowed attention and routed experts does
// between its input projections and its attention, in one launch: routing
// (which reads the layer's input), queries, keys and values, and the
// shared expert's activation max(u, 0)^2.  The three are independent;
// each workgroup does a part of one of them.
#include "router.h"
#include "window_prep.h"

struct SharedAct {
  bf16_t* out;
  const bf16_t* u;
  int ld_out, ld, ff;  // ff 0: there is none
};

// four tokens a prep block; pieces of 8 of ``u`` a thread
#define ACT_PIECES 4
template <int NT, int KQ, int KK>
__global__ __launch_bounds__(256) void window_front_kernel(
    Routing r, WindowPrep p, SharedAct s, int route_blocks, int prep_blocks,
    int act_blocks) {
  extern __shared__ float lds[];
  int b = blockIdx.x;
  if (b < route_blocks) {
    route_block<NT>(r, b, lds);
    return;
  }
  b -= route_blocks;
  if (b < prep_blocks) {
    const int t = b * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
    if (t < p.n_tok) window_prep_wave<bf16_t, KQ, KK>(p, t);
    return;
  }
  b -= prep_blocks;
  const int per_row = s.ff / 8;
  const long long total = (long long)p.n_tok * per_row;
#pragma unroll
  for (int i = 0; i < ACT_PIECES; ++i) {
    const long long id =
        ((long long)i * act_blocks + b) * 256 + threadIdx.x;
    if (id >= total) break;
    const int t = (int)(id / per_row);
    const int c = (int)(id - (long long)t * per_row) * 8;
    float f[8];
    load8(s.u + (size_t)t * s.ld + c, f);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      f[j] = fmaxf(f[j], 0.f);
      f[j] *= f[j];
    }
    store8(s.out + (size_t)t * s.ld_out + c, f);
  }
}

extern "C" {

// 1: done; 0: sizes that take the separate kernels; < 0: an error
int hy_window_front(void* index, void* weight, void* counts, void* pairs,
                    const void* h, const void* w, int width, int E, int top,
                    int groups, int keep, float scale, void* proj, int ld,
                    void* cache, int k_off, int v_off, int H, int G, int D,
                    int V, int rot, const void* wq, const void* wk,
                    const void* cos_sin, float eps, const void* pos,
                    const void* row, const void* bt, int max_blocks,
                    void* act, int ld_act, int u_off, int ff, int n_tok,
                    int dtype, void* stream) {
  const Routing r{(int*)index, (float*)weight, (int*)counts, (int*)pairs, h,
                  w, width, E, top, groups, keep, scale, n_tok};
  const WindowPrep p{proj,
                     cache,
                     (const float*)wq,
                     (const float*)wk,
                     (const float*)cos_sin,
                     (const int*)pos,
                     (const int*)row,
                     (const int*)bt,
                     ld, k_off, v_off, H, G, D, V, rot, max_blocks, n_tok,
                     eps};
  const SharedAct s{(bf16_t*)act, (const bf16_t*)proj + u_off, ld_act, ld,
                    ff};
  if (!routing_ok(r) || !window_prep_ok(p) || ff < 0) return -2;
  if (n_tok <= 0) return 1;
  if (!route_block_ok(r, dtype) || !window_prep_wave_ok(p)) return 0;
  if (ff > 0 && (ff % 8 || ld_act % 8 || u_off % 8 ||
                 ((uintptr_t)act & 15) != 0))
    return 0;
  const int rb = (n_tok + 15) / 16, pb = (n_tok + 3) / 4;
  const long long pieces = (long long)n_tok * (ff / 8);
  const int ab = (int)((pieces + 256 * ACT_PIECES - 1) / (256 * ACT_PIECES));
#define GO(KQ, KK)                                                           \
  hipLaunchKernelGGL((window_front_kernel<NT, KQ, KK>), dim3(rb + pb + ab),  \
                     dim3(256), 4 * route_floats<NT>(E, top, groups),        \
                     (hipStream_t)stream, r, p, s, rb, pb, ab)
  if (E <= 16) {
    constexpr int NT = 1;
    WINDOW_PREP_UNITS(H * D, G * D);
  } else if (E <= 32) {
    constexpr int NT = 2;
    WINDOW_PREP_UNITS(H * D, G * D);
  } else {
    constexpr int NT = 4;
    WINDOW_PREP_UNITS(H * D, G * D);
  }
#undef GO
  HY_CHECK();
  return 1;
}

}  // extern "C"
