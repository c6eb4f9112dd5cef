// kh_scan.h — selective scan:  S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n ;  y_c = sum_n S[c, n] C_n + D_c x_c ;
// out = y silu(z).  fp32 throughout; the state of a sequence stays in its slot between calls.
//
// A lane owns KH_SCAN_NS states of one channel, G = 2^g lanes share a channel (their partial y meet in a DPP
// reduction), 256 / G channels per workgroup.  Prompts are cut into CHUNKS of up to KH_SCAN_CH tokens that run side by
// side:  k_scan_ends  computes every chunk's end state from a zero start and its sum of dt (the chunk's decay is
// exp(A sum dt));  k_scan_carry  walks the chunks of a segment and turns the end states into start states;
// k_scan_out  runs each chunk from its start state, writes the outputs and, in a segment's last chunk, the slot's
// state.  Segments of one chunk (and decoding) need k_scan_out only.
#pragma once
#include "kh_lops.h"

#define KH_SCAN_NS 8
#define KH_SCAN_CH 64
#define KH_SCAN_MAX_STATE 256  // 32 lanes x 8

namespace khm {

struct ScanChunk {
  int seg, row0, n, flags;  // flags: 1 = first of its segment, 2 = last of its segment
};

template <class T>
struct ScanArgs {
  const T* x;            // [T][ldx] convolved inputs
  const T* z;            // [T][ldz] gate (nullptr in k_scan_ends)
  const float* dt;       // [T][C]
  const float* bc;       // [T][2 N]: B then C
  const float *A2, *D;   // A2 = -exp(A_log) log2(e)  [C][N], D [C]
  T* out;                // [T][ldo]
  float* state;          // + slot * slot_stride: [C][N]
  size_t slot_stride;
  float *ends, *dtsum;   // [chunks][C][N], [chunks][C]
  const ScanChunk* chunks;
  PassTabs p;
  int C, N, ldx, ldz, ldo, gshift;
};

template <int G>
__device__ __forceinline__ float scan_group_sum(float v) { return group_sum<G>(v); }

// B and C rows of the chunk go to LDS: [n_tok][2 N]
template <class T, bool OUT, int G>
__global__ __launch_bounds__(256) void k_scan(const ScanArgs<T> a) {
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  float* bc = (float*)smem_raw;
  const ScanChunk ck = a.chunks[blockIdx.y];
  if (!OUT && (ck.flags & 2)) return;  // nobody continues from a last chunk's zero-start end
  const int N = a.N, NP = G * KH_SCAN_NS;  // LDS rows padded to whole lanes
  for (int i = threadIdx.x; i < ck.n * NP * 2; i += 256) {
    const int t = i / (2 * NP), r = i - t * (2 * NP), which = r >= NP, n = r - which * NP;
    bc[i] = n < N ? a.bc[(size_t)(ck.row0 + t) * (2 * N) + which * N + n] : 0.f;
  }
  __syncthreads();
  const int g = threadIdx.x & (G - 1);
  const int c = blockIdx.x * (256 / G) + (int)threadIdx.x / G;
  const bool live = c < a.C;
  const int cc = live ? c : a.C - 1;
  const int n0 = g * KH_SCAN_NS;
  float A2[KH_SCAN_NS], S[KH_SCAN_NS];
  const size_t sbase = (size_t)cc * N;
  const bool first = ck.flags & 1;
  const int slot = a.p.seg_slot[ck.seg];
  float* st = a.state + (size_t)slot * a.slot_stride + sbase;
  const bool fresh = a.p.seg_pos0[ck.seg] == 0;
#pragma unroll
  for (int j = 0; j < KH_SCAN_NS; ++j) {
    const int n = n0 + j;
    A2[j] = n < N ? a.A2[sbase + n] : 0.f;
    S[j] = 0.f;
    if (OUT && n < N) {
      if (!first) S[j] = a.ends[(size_t)blockIdx.y * a.C * N + sbase + n];  // start state (k_scan_carry)
      else if (!fresh) S[j] = st[n];
    }
  }
  const float D = OUT ? a.D[cc] : 0.f;
  float dts = 0.f;
  const T* xp = a.x + (size_t)ck.row0 * a.ldx + cc;
  const float* dp = a.dt + (size_t)ck.row0 * a.C + cc;
  const T* zp = OUT ? a.z + (size_t)ck.row0 * a.ldz + cc : nullptr;
  constexpr int U = 4;  // tokens requested together
  for (int t0 = 0; t0 < ck.n; t0 += U) {
    float xv[U], dv[U], zv[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int t = t0 + u < ck.n ? t0 + u : ck.n - 1;
      xv[u] = (float)xp[(size_t)t * a.ldx];
      dv[u] = dp[(size_t)t * a.C];
      zv[u] = OUT ? (float)zp[(size_t)t * a.ldz] : 0.f;
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (t0 + u >= ck.n) break;
      const float* b = bc + (size_t)(t0 + u) * 2 * NP + n0;
      const float dx = dv[u] * xv[u];
      float y = 0.f;
#pragma unroll
      for (int j = 0; j < KH_SCAN_NS; ++j) {
        S[j] = __builtin_fmaf(__builtin_amdgcn_exp2f(dv[u] * A2[j]), S[j], dx * b[j]);
        if (OUT) y = __builtin_fmaf(S[j], b[NP + j], y);
      }
      dts += dv[u];
      if (OUT) {
        y = scan_group_sum<G>(y);
        y = __builtin_fmaf(D, xv[u], y);
        if (g == 0 && live) a.out[(size_t)(ck.row0 + t0 + u) * a.ldo + c] = (T)(y * silu1(zv[u]));
      }
    }
  }
  if (!live) return;
#pragma unroll
  for (int j = 0; j < KH_SCAN_NS; ++j) {
    const int n = n0 + j;
    if (n >= N) continue;
    if (OUT) {
      if (ck.flags & 2) st[n] = S[j];
    } else {
      a.ends[(size_t)blockIdx.y * a.C * N + sbase + n] = S[j];
    }
  }
  if (!OUT && g == 0) a.dtsum[(size_t)blockIdx.y * a.C + c] = dts;
}

// ends[k] (end of chunk k from zero) -> start state of chunk k, for every segment's chunks in order.
// grid (C N / 256, segments with more than one chunk); chunk0 / nchunk per such segment
template <class T>
__global__ __launch_bounds__(256) void k_scan_carry(const ScanArgs<T> a, const int32_t* chunk0, const int32_t* nchunk) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x, CN = (size_t)a.C * a.N;
  if (i >= CN) return;
  const int k0 = chunk0[blockIdx.y], nk = nchunk[blockIdx.y];
  const int seg = a.chunks[k0].seg;
  const float A2 = a.A2[i];
  const int c = (int)(i / a.N);
  float S = a.p.seg_pos0[seg] == 0 ? 0.f : a.state[(size_t)a.p.seg_slot[seg] * a.slot_stride + i];
  for (int k = k0; k < k0 + nk; ++k) {
    const float e = k + 1 < k0 + nk ? a.ends[(size_t)k * CN + i] : 0.f;
    a.ends[(size_t)k * CN + i] = S;
    if (k + 1 < k0 + nk) S = __builtin_fmaf(__builtin_amdgcn_exp2f(A2 * a.dtsum[(size_t)k * a.C + c]), S, e);
  }
}

template <class T, bool OUT>
int scan_launch(hipStream_t s, const ScanArgs<T>& a, int nchunks) {
  int G = 1;
  while (G * KH_SCAN_NS < a.N) G <<= 1;
  const dim3 grid((a.C + 256 / G - 1) / (256 / G), nchunks);
  const size_t lds = (size_t)KH_SCAN_CH * 2 * G * KH_SCAN_NS * 4;
  auto go = [&](auto kern) -> int {
    if (lds > 64 * 1024 &&
        hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
      return KH_ERR_UNSUPPORTED;
    hipLaunchKernelGGL(kern, grid, dim3(256), lds, s, a);
    return KH_OK;
  };
  switch (G) {
    case 1: return go(k_scan<T, OUT, 1>);
    case 2: return go(k_scan<T, OUT, 2>);
    case 4: return go(k_scan<T, OUT, 4>);
    case 8: return go(k_scan<T, OUT, 8>);
    case 16: return go(k_scan<T, OUT, 16>);
    case 32: return go(k_scan<T, OUT, 32>);
    default: return KH_ERR_UNSUPPORTED;
  }
}
}  // namespace khm
