// kh_lops.h — per-token kernels of the layer-list models: embedding, the residual update fused with the two layer
// norms of a parallel block, the causal convolution.  Everything that touches the residual stream is fp32.
#pragma once
#include "kh_tile.h"

namespace khm {

// Tables of one pass: T tokens of up to S sequences, concatenated.  All arrays live on the device.
struct PassTabs {
  const int32_t *tok, *pos, *seg;              // [T]: token id, position in its sequence, segment
  const int32_t *seg_slot, *seg_row0, *seg_n, *seg_pos0;  // [S]: state slot, first row, rows, position of the first row
};

// what one layer leaves to be added to the residual stream
struct AddArgs {
  const float* mix;       // [T][W] mixer output (nullptr: nothing pending)
  // experts: sum_k w[t][k] y[slot[t][k]] (slot < 0: not a stored row), identity weight, gated shared expert
  const float* y;         // expert output rows [rows][W]
  const int32_t* y_slot;  // [T][top]
  const float* y_w;       // [T][top]
  const float* id_w;      // [T]
  const float* sh;        // [T][W] shared expert's output
  const float* sh_g;      // [T] its gate
  int top;
};

// One workgroup per token.  x += pending; (loop entry) x += x0, x += step; then xn1 / xn2 = layer norms of x.
// x_src: 0 = x itself, 1 = the embedding row (first layer; also fills x0).
template <class T>
struct CombineArgs {
  float *x, *x0;
  AddArgs add;
  const T* embed;
  const int32_t* tok;
  const float* step;                       // [W] or nullptr
  const float *w1, *b1, *w2, *b2;          // norm parameters (w1 nullptr: no norm output)
  T *xn1, *xn2;                            // [T][ld]
  const T* xn2_prev;                       // identity experts' input: the xn2 the pending layer read
  int W, ld, from_embed, add_x0;
  float eps;
};
template <class T>
__global__ __launch_bounds__(256) void k_combine(const CombineArgs<T> a) {
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  float* row = (float*)smem_raw;
  __shared__ float red[KH_WAVES_MAX];
  const int t = blockIdx.x;
  const size_t o = (size_t)t * a.W;
  float* x = a.x + o;
  float s = 0.f;
  const T* e = a.from_embed ? a.embed + (size_t)a.tok[t] * a.W : nullptr;
  float idw = 0.f, shg = 0.f;
  const int top = a.add.y ? a.add.top : 0;
  if (a.add.y) {
    idw = a.add.id_w[t];
    shg = a.add.sh ? a.add.sh_g[t] : 0.f;
  }
  for (int i = threadIdx.x; i < a.W; i += 256) {
    float v;
    if (a.from_embed) {
      v = (float)e[i];
      a.x0[o + i] = v;
    } else {
      v = x[i];
    }
    if (a.add.mix) {
      float d = a.add.mix[o + i];
      if (a.add.y) {
        float f = 0.f;
        for (int k = 0; k < top; ++k) {
          const int sl = a.add.y_slot[(size_t)t * top + k];
          if (sl >= 0) f = __builtin_fmaf(a.add.y_w[(size_t)t * top + k], a.add.y[(size_t)sl * a.W + i], f);
        }
        if (idw != 0.f) f = __builtin_fmaf(idw, (float)a.xn2_prev[(size_t)t * a.ld + i], f);
        if (a.add.sh) f = __builtin_fmaf(shg, a.add.sh[o + i], f);
        d += f;
      }
      v += d;
    }
    if (a.add_x0) v += a.x0[o + i];
    if (a.step) v += a.step[i];
    x[i] = v;
    row[i] = v;
    s += v;
  }
  if (!a.w1) return;
  const float mean = block_sum(s, red) / (float)a.W;
  float q = 0.f;
  for (int i = threadIdx.x; i < a.W; i += 256) {
    const float d = row[i] - mean;
    q = __builtin_fmaf(d, d, q);
  }
  const float rstd = 1.0f / sqrtf(block_sum(q, red) / (float)a.W + a.eps);
  for (int i = threadIdx.x; i < a.W; i += 256) {
    const float n = (row[i] - mean) * rstd;
    a.xn1[(size_t)t * a.ld + i] = (T)(n * a.w1[i] + a.b1[i]);
    if (a.w2) a.xn2[(size_t)t * a.ld + i] = (T)(n * a.w2[i] + a.b2[i]);
  }
}

// layer norm of gathered rows: out[r] = norm(x[rows[r]])
template <class T>
__global__ __launch_bounds__(256) void k_gather_norm(const float* x, const int32_t* rows, const float* w, const float* b,
                                                     T* out, int W, int ld, float eps) {
  __shared__ float red[KH_WAVES_MAX];
  const float* r = x + (size_t)rows[blockIdx.x] * W;
  float s = 0.f;
  for (int i = threadIdx.x; i < W; i += 256) s += r[i];
  const float mean = block_sum(s, red) / (float)W;
  float q = 0.f;
  for (int i = threadIdx.x; i < W; i += 256) {
    const float d = r[i] - mean;
    q = __builtin_fmaf(d, d, q);
  }
  const float rstd = 1.0f / sqrtf(block_sum(q, red) / (float)W + eps);
  for (int i = threadIdx.x; i < W; i += 256)
    out[(size_t)blockIdx.x * ld + i] = (T)((r[i] - mean) * rstd * w[i] + b[i]);
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
template <class T>
__global__ __launch_bounds__(256) void k_conv_silu(const ConvArgs<T> a) {
  const int c = blockIdx.x * 256 + threadIdx.x, t = blockIdx.y;
  if (c >= a.C) return;
  const int sg = a.p.seg[t], i = t - a.p.seg_row0[sg];
  const bool fresh = a.p.seg_pos0[sg] == 0;
  const float* st = a.state + (size_t)a.p.seg_slot[sg] * a.slot_stride;
  float v = a.b[c];
  for (int k = 0; k < a.taps; ++k) {
    const int j = i - (a.taps - 1) + k;  // row of the segment
    float in = 0.f;
    if (j >= 0) in = (float)a.xz[(size_t)(t - i + j) * a.ldx + c];
    else if (!fresh) in = st[(size_t)(a.taps - 1 + j) * a.C + c];
    v = __builtin_fmaf(a.w[(size_t)c * a.taps + k], in, v);
  }
  a.out[(size_t)t * a.ldo + c] = (T)silu1(v);
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
