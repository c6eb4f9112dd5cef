// kh_lops.h — per-token kernels of the layer-list models: embedding, the residual update fused with the one or two norms
// of a parallel block (layer norm or RMS norm), the causal convolution.  Everything that touches the residual stream is fp32.
#pragma once
#include "kh_tile.h"

namespace khm {

// Tables of one pass: T tokens of up to S sequences, concatenated.  All arrays live on the device.
struct PassTabs {
  const int32_t *tok, *pos, *seg;              // [T]: token id, position in its sequence, segment
  const int32_t *seg_slot, *seg_row0, *seg_n, *seg_pos0;  // [S]: state slot, first row, rows, position of the first row
};

// what one layer leaves to be added to the residual stream
template <class T>
struct AddArgs {
  const float* mix;       // [T][ld] mixer output (nullptr: nothing pending)
  // experts: sum_k w[t][k] y[slot[t][k]] (slot < 0: not a stored row), identity weight, gated shared expert
  const T* y;             // expert output rows [rows][ld]
  const int32_t* y_slot;  // [T][top]
  const float* y_w;       // [T][top]
  const float* id_w;      // [T]
  const T* sh;            // [T][ld] shared expert's output
  const float* sh_g;      // [T] its gate (nullptr: 1)
  int top;
};

// One workgroup per token.  x += mult * pending; (loop entry) x += x0, x += step; then xn1 / xn2 = norms of x, or
// cat = [x | x0] for a loop that enters through a matrix.  The embedding output is scale * embed[token] + pos[position].
// Rows of every array are ld (a multiple of KH_LPAD) elements with zeros behind the W valid ones.
template <class T>
struct CombineArgs {
  float *x, *x0;
  AddArgs<T> add;
  const T *embed, *pos_emb;                // pos_emb nullptr: none
  const int32_t *tok, *pos;
  const float* step;                       // one row or nullptr
  const float *w1, *b1, *w2, *b2;          // norm parameters (w1 nullptr: no norm output)
  T *xn1, *xn2;
  T* cat;                                  // [T][2 ld] or nullptr
  const T* xn2_prev;                       // identity experts' input: the xn2 the pending layer read
  int W, ld, from_embed, add_x0, rms;      // rms: no mean, biases may be nullptr
  float eps, mult, emb_scale;
};
template <class T>
__device__ __forceinline__ f32x4 quad_f(const T* p) {
  const typename Tile<T>::quad q = *(const typename Tile<T>::quad*)p;
  return f32x4{(float)q.x, (float)q.y, (float)q.z, (float)q.w};
}
__device__ __forceinline__ f32x4 fma_s(float s, f32x4 a, f32x4 b) {
  f32x4 r;
#pragma unroll
  for (int i = 0; i < 4; ++i) r[i] = __builtin_fmaf(s, a[i], b[i]);
  return r;
}
template <class T>
__global__ __launch_bounds__(256) void k_combine(const CombineArgs<T> a) {
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  f32x4* row = (f32x4*)smem_raw;  // [ld / 4]
  __shared__ float red[KH_WAVES_MAX];
  const int t = blockIdx.x, n4 = a.ld >> 2;
  const size_t o = (size_t)t * a.ld;
  float s = 0.f;
  const T* e = a.from_embed ? a.embed + (size_t)a.tok[t] * a.ld : nullptr;
  const T* ep = a.from_embed && a.pos_emb ? a.pos_emb + (size_t)a.pos[t] * a.ld : nullptr;
  const float idw = a.add.y && a.add.id_w ? a.add.id_w[t] : 0.f, shg = a.add.sh && a.add.sh_g ? a.add.sh_g[t] : 1.f;
  const int top = a.add.y ? a.add.top : 0;
  for (int i = threadIdx.x; i < n4; i += 256) {
    const int c = 4 * i;
    f32x4 v;
    if (a.from_embed) {
      v = quad_f(e + c) * a.emb_scale;
      if (ep) v += quad_f(ep + c);
      *(f32x4*)(a.x0 + o + c) = v;
    } else {
      v = *(const f32x4*)(a.x + o + c);
    }
    if (a.add.mix) {
      f32x4 d = *(const f32x4*)(a.add.mix + o + c);
      f32x4 f = {0.f, 0.f, 0.f, 0.f};
      for (int k = 0; k < top; ++k) {
        const int sl = a.add.y_slot[(size_t)t * top + k];
        if (sl >= 0) f = fma_s(a.add.y_w[(size_t)t * top + k], quad_f(a.add.y + (size_t)sl * a.ld + c), f);
      }
      if (idw != 0.f) f = fma_s(idw, quad_f(a.xn2_prev + o + c), f);
      if (a.add.sh) f = fma_s(shg, quad_f(a.add.sh + o + c), f);
      d += f;
      v = fma_s(a.mult, d, v);
    }
    if (a.add_x0) v += *(const f32x4*)(a.x0 + o + c);
    if (a.step) v += *(const f32x4*)(a.step + c);
    *(f32x4*)(a.x + o + c) = v;
    if (a.cat) {
      *(typename Tile<T>::quad*)(a.cat + 2 * o + c) = to_quad<T>(v);
      *(typename Tile<T>::quad*)(a.cat + 2 * o + a.ld + c) = to_quad<T>(a.from_embed ? v : *(const f32x4*)(a.x0 + o + c));
    }
    row[i] = v;
    s += (v.x + v.y) + (v.z + v.w);
  }
  if (!a.w1) return;
  const float mean = a.rms ? 0.f : block_sum(s, red) / (float)a.W;
  float q = 0.f;
  for (int i = threadIdx.x; i < n4; i += 256) {
    const f32x4 v = row[i];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const float d = 4 * i + k < a.W ? v[k] - mean : 0.f;
      q = __builtin_fmaf(d, d, q);
    }
  }
  const float rstd = 1.0f / sqrtf(block_sum(q, red) / (float)a.W + a.eps);
  for (int i = threadIdx.x; i < n4; i += 256) {
    const int c = 4 * i;
    const f32x4 v = row[i];
    f32x4 y;
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    const f32x4 w1 = *(const f32x4*)(a.w1 + c), b1 = a.b1 ? *(const f32x4*)(a.b1 + c) : zero;
#pragma unroll
    for (int k = 0; k < 4; ++k) y[k] = (v[k] - mean) * rstd * w1[k] + b1[k];  // pads: weights and biases are zero
    *(typename Tile<T>::quad*)(a.xn1 + o + c) = to_quad<T>(y);
    if (a.w2) {
      const f32x4 w2 = *(const f32x4*)(a.w2 + c), b2 = a.b2 ? *(const f32x4*)(a.b2 + c) : zero;
#pragma unroll
      for (int k = 0; k < 4; ++k) y[k] = (v[k] - mean) * rstd * w2[k] + b2[k];
      *(typename Tile<T>::quad*)(a.xn2 + o + c) = to_quad<T>(y);
    }
  }
}

// norm of gathered rows: out[r] = norm(x[rows[r]]); rows of ld elements on both sides.  rms: no mean, b may be nullptr
template <class T>
__global__ __launch_bounds__(256) void k_gather_norm(const float* x, const int32_t* rows, const float* w, const float* b,
                                                     T* out, int W, int ld, float eps, int rms) {
  __shared__ float red[KH_WAVES_MAX];
  const float* r = x + (size_t)rows[blockIdx.x] * ld;
  float s = 0.f;
  for (int i = threadIdx.x; i < W; i += 256) s += r[i];
  const float mean = rms ? 0.f : block_sum(s, red) / (float)W;
  float q = 0.f;
  for (int i = threadIdx.x; i < W; i += 256) {
    const float d = r[i] - mean;
    q = __builtin_fmaf(d, d, q);
  }
  const float rstd = 1.0f / sqrtf(block_sum(q, red) / (float)W + eps);
  for (int i = threadIdx.x; i < W; i += 256)
    out[(size_t)blockIdx.x * ld + i] = (T)((r[i] - mean) * rstd * w[i] + (b ? b[i] : 0.f));
}

// ---- causal depthwise convolution + silu -----------------------------------------------------------------------
// Inputs are the first C columns of xz rows.  Inputs before a segment's first row come from the sequence's conv state
// [taps - 1][C] (position 0: zeros).  grid (C / 256, T).
template <class T>
struct ConvArgs {
  const T* xz;          // [T][ldx]
  T* out;               // [T][ldo]
  const float *w, *b;   // [C][taps], [C]
  float* state;         // + slot * slot_stride
  size_t slot_stride;
  int C, ldx, ldo, taps;
  PassTabs p;
};
// E channels (16 bytes) of KH_CONV_TT consecutive tokens per thread; the taps of the channels stay in registers.
// TAPS: number of taps, 0 = any (weights re-read per token).  grid (C / (256 E), T / KH_CONV_TT)
#define KH_CONV_TT 8
template <class T, int TAPS>
__global__ __launch_bounds__(256) void k_conv_silu(const ConvArgs<T> a, int T_all) {
  constexpr int E = Tile<T>::N;
  typedef typename Tile<T>::frag frag;
  const int c = (blockIdx.x * 256 + threadIdx.x) * E;
  if (c >= a.C) return;
  const bool vec = c + E <= a.C && (a.ldx & (E - 1)) == 0;
  const int taps = TAPS ? TAPS : a.taps;
  float w[E][TAPS ? TAPS : 1], bias[E];
#pragma unroll
  for (int e = 0; e < E; ++e) {
    bias[e] = c + e < a.C ? a.b[c + e] : 0.f;
    if (TAPS)
#pragma unroll
      for (int k = 0; k < TAPS; ++k) w[e][k] = c + e < a.C ? a.w[(size_t)(c + e) * TAPS + k] : 0.f;
  }
  for (int u = 0; u < KH_CONV_TT; ++u) {
    const int t = blockIdx.y * KH_CONV_TT + u;
    if (t >= T_all) return;
    const int sg = a.p.seg[t], i = t - a.p.seg_row0[sg];
    float v[E];
#pragma unroll
    for (int e = 0; e < E; ++e) v[e] = bias[e];
    auto tap = [&](int k, const float (&in)[E]) __attribute__((always_inline)) {
#pragma unroll
      for (int e = 0; e < E; ++e)
        v[e] = __builtin_fmaf(TAPS ? w[e][TAPS ? k : 0] : (c + e < a.C ? a.w[(size_t)(c + e) * taps + k] : 0.f), in[e], v[e]);
    };
    auto from_row = [&](int j, float (&in)[E]) __attribute__((always_inline)) {
      const T* x = a.xz + (size_t)(t - i + j) * a.ldx + c;
      if (vec) {
        const frag f = *(const frag*)x;
#pragma unroll
        for (int e = 0; e < E; ++e) in[e] = (float)f[e];
      } else {
#pragma unroll
        for (int e = 0; e < E; ++e) in[e] = c + e < a.C ? (float)x[e] : 0.f;
      }
    };
    float in[E];
    if (i >= taps - 1) {  // every input is a row of the segment
      if (TAPS) {
#pragma unroll
        for (int k = 0; k < TAPS; ++k) {
          from_row(i - (TAPS - 1) + k, in);
          tap(k, in);
        }
      } else {
        for (int k = 0; k < taps; ++k) {
          from_row(i - (taps - 1) + k, in);
          tap(k, in);
        }
      }
    } else {
      const bool fresh = a.p.seg_pos0[sg] == 0;
      const float* st = a.state + (size_t)a.p.seg_slot[sg] * a.slot_stride;
      auto edge = [&](int k) __attribute__((always_inline)) {
        const int j = i - (taps - 1) + k;
        if (j >= 0) {
          from_row(j, in);
        } else {
#pragma unroll
          for (int e = 0; e < E; ++e) in[e] = !fresh && c + e < a.C ? st[(size_t)(taps - 1 + j) * a.C + c + e] : 0.f;
        }
        tap(k, in);
      };
      if constexpr (TAPS != 0) {
#pragma unroll
        for (int k = 0; k < TAPS; ++k) edge(k);
      } else {
        for (int k = 0; k < taps; ++k) edge(k);
      }
    }
    frag f;  // output rows are padded to whole fragments
#pragma unroll
    for (int e = 0; e < E; ++e) f[e] = (T)(c + e < a.C ? silu1(v[e]) : 0.f);
    *(frag*)(a.out + (size_t)t * a.ldo + c) = f;
  }
}
template <class T>
void conv_launch(hipStream_t s, const ConvArgs<T>& a, int T_all) {
  constexpr int CW = 256 * Tile<T>::N;
  const dim3 g((a.C + CW - 1) / CW, (T_all + KH_CONV_TT - 1) / KH_CONV_TT);
  if (a.taps == 4) hipLaunchKernelGGL((k_conv_silu<T, 4>), g, dim3(256), 0, s, a, T_all);
  else hipLaunchKernelGGL((k_conv_silu<T, 0>), g, dim3(256), 0, s, a, T_all);
}
// the last taps - 1 inputs of every segment become its sequence's state.  grid (C / 256, S)
template <class T>
__global__ __launch_bounds__(256) void k_conv_state(const ConvArgs<T> a) {
  const int c = blockIdx.x * 256 + threadIdx.x, sg = blockIdx.y;
  if (c >= a.C) return;
  const int n = a.p.seg_n[sg], row0 = a.p.seg_row0[sg], m = a.taps - 1;
  const bool fresh = a.p.seg_pos0[sg] == 0;
  float* st = a.state + (size_t)a.p.seg_slot[sg] * a.slot_stride;
  for (int j = 0; j < m; ++j) {  // ascending: entry j reads entry j + n > j of the old state
    const int i = n - m + j;
    float v = 0.f;
    if (i >= 0) v = (float)a.xz[(size_t)(row0 + i) * a.ldx + c];
    else if (!fresh) v = st[(size_t)(j + n) * a.C + c];
    st[(size_t)j * a.C + c] = v;
  }
}
}  // namespace khm
