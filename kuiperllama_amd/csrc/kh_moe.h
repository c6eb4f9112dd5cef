// kh_moe.h — expert router and dispatch lists.
// Two forms, both fp32, ties to the lower index:
//   over all     scores s = softmax(z) over all router outputs; the `top` largest s + correction are chosen; the weights
//                are the chosen s
//   over chosen  the `top` largest z are chosen; the weights are the softmax over them alone
// Outputs from n_expert on are identity experts (no tensors).
#pragma once
#include "kh_lgemm.h"

#define KH_MOE_MAX_OUT 1024  // router outputs (16 per lane)
#define KH_MOE_MAX_TOP 32

namespace khm {

// The choice for one token by one wave; z in LDS or global [n_out], n_out <= 64 PER.  Calls pick(k, id, weight) for
// k = 0 .. top - 1 on every lane with wave-uniform values, in order of decreasing choice score.  Weights are to be
// multiplied by the returned factor.  corr nullptr: none.
template <int PER, class F>
__device__ __forceinline__ float moe_route(const float* z, const float* corr, int n_out, int top, bool over_chosen, int lane,
                                           F&& pick) {
  float s[PER], key[PER];
  float m = -INFINITY;
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int i = j * 64 + lane;
    s[j] = i < n_out ? z[i] : -INFINITY;
    key[j] = corr && i < n_out ? corr[i] : 0.f;
    m = fmaxf(m, s[j]);
  }
  m = wave_max(m);
  float sum = 0.f;
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    if (over_chosen) key[j] = s[j];
    s[j] = expf(s[j] - m);  // exp(-inf) = 0 beyond n_out
    sum += s[j];
  }
  if (!over_chosen) {
    sum = wave_sum(sum);
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      s[j] /= sum;
      key[j] = j * 64 + lane < n_out ? s[j] + key[j] : -INFINITY;
    }
  }
  float chosen = 0.f;
  for (int k = 0; k < top; ++k) {
    float v = key[0];
#pragma unroll
    for (int j = 1; j < PER; ++j) v = fmaxf(v, key[j]);
    v = wave_max(v);
    // lowest index that holds the maximum (indices are exact in fp32)
    float first = 1e9f;
#pragma unroll
    for (int j = PER - 1; j >= 0; --j) first = key[j] == v ? (float)(j * 64 + lane) : first;
    const int id = (int)(-wave_max(-first));
    float w = 0.f;
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const bool mine = j * 64 + lane == id;
      w = mine ? s[j] : w;
      key[j] = mine ? -INFINITY : key[j];
    }
    w = wave_sum(w);  // one lane holds it, the others zero
    chosen += w;
    pick(k, __builtin_amdgcn_readfirstlane(id), w);
  }
  return over_chosen ? 1.0f / chosen : 1.0f;  // the largest z contributes exp(0)
}

struct RouteArgs {
  const float* z;        // [T][ldz]: router outputs, then (shared expert) its gate logit
  const float* corr;     // [n_out] or nullptr
  int32_t* id;           // [T][top]
  float* w;              // [T][top]
  float* id_w;           // [T] summed weight of the chosen identity experts
  float* sh_g;           // [T] sigmoid of the shared expert's gate
  int T, ldz, n_out, n_expert, top, shared, over_chosen;
};
template <int PER>
__global__ __launch_bounds__(256) void k_moe_route(const RouteArgs a) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (t >= a.T) return;
  const float* z = a.z + (size_t)t * a.ldz;
  float idw = 0.f, my_w = 0.f;
  int my_id = 0;
  const float f = moe_route<PER>(z, a.corr, a.n_out, a.top, a.over_chosen, lane, [&](int k, int id, float w) __attribute__((always_inline)) {
    if (id >= a.n_expert) idw += w;
    my_id = lane == k ? id : my_id;  // top <= KH_MOE_MAX_TOP < 64: lane k keeps choice k
    my_w = lane == k ? w : my_w;
  });
  if (lane < a.top) {
    a.id[(size_t)t * a.top + lane] = my_id;
    a.w[(size_t)t * a.top + lane] = my_w * f;
  }
  if (lane == 0) {
    a.id_w[t] = idw * f;
    if (a.shared) a.sh_g[t] = sigmoid1(z[a.n_out]);
  }
}

static inline int moe_per(int n_out) { return n_out <= 64 ? 1 : (n_out <= 256 ? 4 : 16); }
static inline void moe_route_launch(hipStream_t s, const RouteArgs& a) {
  const dim3 g((a.T + 3) / 4), b(256);
  const int per = moe_per(a.n_out);
  if (per == 1) hipLaunchKernelGGL(k_moe_route<1>, g, b, 0, s, a);
  else if (per == 4) hipLaunchKernelGGL(k_moe_route<4>, g, b, 0, s, a);
  else hipLaunchKernelGGL(k_moe_route<16>, g, b, 0, s, a);
}

// Dispatch lists, one workgroup: rows grouped by expert (row -> token), slot of every (token, choice) in that order
// (-1: identity expert), and the token tiles of the grouped GEMMs.
struct ListArgs {
  const int32_t* id;  // [T][top]
  int32_t *rows, *slot;
  LgTile* tiles;
  int32_t* n_tiles;
  int T, top, n_expert, bm;
};
static __global__ __launch_bounds__(1024) void k_moe_lists(const ListArgs a) {
  __shared__ int32_t cnt[KH_MOE_MAX_OUT], off[KH_MOE_MAX_OUT], tile[KH_MOE_MAX_OUT];
  for (int e = threadIdx.x; e < a.n_expert; e += 1024) cnt[e] = 0;
  __syncthreads();
  const int n = a.T * a.top;
  for (int i = threadIdx.x; i < n; i += 1024) {
    const int e = a.id[i];
    if (e < a.n_expert) atomicAdd(&cnt[e], 1);
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    int o = 0, q = 0;
    for (int e = 0; e < a.n_expert; ++e) {
      off[e] = o;
      tile[e] = q;
      o += cnt[e];
      q += (cnt[e] + a.bm - 1) / a.bm;
    }
    *a.n_tiles = q;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < a.n_expert; e += 1024) {
    const int c = cnt[e];
    for (int r = 0, q = tile[e]; r < c; r += a.bm, ++q) a.tiles[q] = LgTile{e, off[e] + r, c - r < a.bm ? c - r : a.bm, 0};
  }
  __syncthreads();
  for (int i = threadIdx.x; i < n; i += 1024) {
    const int e = a.id[i];
    int p = -1;
    if (e < a.n_expert) {
      p = atomicAdd(&off[e], 1);
      a.rows[p] = i / a.top;
    }
    a.slot[i] = p;
  }
}
}  // namespace khm
