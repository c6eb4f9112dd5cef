// kh_ldecode.h — fused decode step of the layer-list models: B sequences (1, 2 or 4), one token each.
//
// Per layer   mixer mamba1: 4 launches      latent attention: 6      attention over heads: 5
//   k_ld_in   norms -> LDS ; every projection that reads them: mixer input (+ bias), router (+ shared gate row), dense
//             or shared feed-forward's gate / up ; mamba x rows go through the convolution and silu in the epilogue
//   k_ld_mid  router choice, chosen experts' gate / up ; mamba: W_x ; latent: W_uq behind its RMS norm, cache row ;
//             heads: cache row
//   mamba     k_ld_scan   dt projection, softplus, one step of the selective scan, gate
//   latent    k_ld_absorb W_uk^T q per head, rotation ; k_latent_attn (time splits) ; k_ld_values merge + W_uv per head
//   heads     k_heads_attn (time splits) ; k_ld_merge merge and output gate
//   k_ld_out  W_o . v (+ bias) + experts' down + shared down + identity experts, times the residual multiplier, +
//             residual: one dot product per row over a concatenation of weight rows
// A loop that enters through a matrix: k_ld_enter in front of each pass.  Then k_ld_head (final norm, head, soft cap,
// argmax partials) and the sampler of kh_fused.h.
//
// GEMV core: a wave owns R rows.  A row is cut into BLOCKS of 64 x 16 bytes; U blocks of R rows are requested together
// (non-temporal), and the first tile of a wave is requested before the input vectors are staged.  Vectors lie in LDS
// as fp32, block by block, split into planes of four so that a lane's reads are consecutive 16-byte slots; their tails
// are zeros, so the clamped weight loads of a tail lane contribute nothing.  Accumulation is fp32.
#pragma once
#include "kh_heads.h"
#include "kh_hybrid.h"

namespace khm {

template <class T>
struct Ld {
  static constexpr int E = Tile<T>::N;     // elements of a 16-byte load
  static constexpr int P = E / 4;          // float4 planes of a block
  static constexpr int BE = 64 * E;        // elements of a block
  static __host__ __device__ __forceinline__ int blocks(int n) { return (n + BE - 1) / BE; }
  static __host__ __device__ __forceinline__ size_t vec_bytes(int n) { return (size_t)blocks(n) * BE * 4; }
  // place (in floats) of element i of a staged vector
  static __device__ __forceinline__ int place(int i) {
    const int b = i / BE, r = i - b * BE, l = r / E, e = r - l * E;
    return b * BE + ((e >> 2) * 64 + l) * 4 + (e & 3);
  }
};

// float4 group i (elements 4 i ..) of a staged vector: its 16-byte slot
template <class T>
__device__ __forceinline__ int ld_slot(int i) {
  constexpr int B4 = Ld<T>::BE / 4, P = Ld<T>::P;
  const int b = i / B4, r = i - b * B4;
  return b * B4 + (r % P) * 64 + r / P;
}
__device__ __forceinline__ f32x4 f4_zero() { return f32x4{0.f, 0.f, 0.f, 0.f}; }
// n4 valid float4 of src -> slots [0, total4), zeros behind them; times g
template <class T, int NT>
__device__ __forceinline__ void ld_stage(f32x4* xs, const float* src, int n4, int total4, float g, int tid) {
  for (int i0 = tid; i0 < total4; i0 += 4 * NT) {
    f32x4 v[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int i = i0 + j * NT;
      v[j] = i < n4 ? ((const f32x4*)src)[i] : f4_zero();
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (i0 + j * NT < total4) xs[ld_slot<T>(i0 + j * NT)] = v[j] * g;
  }
}
// Layer norm (rms: RMS norm, shift 0) of one row (256 threads, NV float4 each, rows padded with zeros to ld) into LDS
// slots.  v: the row in registers; returns the normalised values in v (also written to `out` when given).  Mean and
// variance come from ONE workgroup reduction of (x - shift) and (x - shift)^2, shift = an element of the row: no
// cancellation beyond the distance of that element from the mean.  red: 2 KH_WAVES_MAX floats.
template <class T, int NV>
__device__ __forceinline__ void ld_norm(f32x4 (&v)[NV], const f32x4 (&w)[NV], const f32x4 (&b)[NV], float shift, bool rms, int W,
                                        int n4, int total4, float eps, float* red, f32x4* xs, f32x4* out) {
  float s1 = 0.f, s2 = 0.f;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int i = threadIdx.x + 256 * j;
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const float d = 4 * i + k < W ? v[j][k] - shift : 0.f;
      s1 += d;
      s2 = __builtin_fmaf(d, d, s2);
    }
  }
  s1 = wave_sum(s1);
  s2 = wave_sum(s2);
  const int wave = threadIdx.x >> 6;
  if ((threadIdx.x & 63) == 0) {
    red[wave] = s1;
    red[KH_WAVES_MAX + wave] = s2;
  }
  __syncthreads();
  s1 = (red[0] + red[1]) + (red[2] + red[3]);
  s2 = (red[KH_WAVES_MAX] + red[KH_WAVES_MAX + 1]) + (red[KH_WAVES_MAX + 2] + red[KH_WAVES_MAX + 3]);
  const float m = rms ? 0.f : s1 / (float)W, mean = rms ? 0.f : shift + m;
  const float var = fmaxf(s2 / (float)W - m * m, 0.f);
  const float rstd = 1.0f / sqrtf(var + eps);
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int i = threadIdx.x + 256 * j;
#pragma unroll
    for (int k = 0; k < 4; ++k) v[j][k] = (v[j][k] - mean) * rstd * w[j][k] + b[j][k];  // pads: zero weight and bias
    if (i < total4) xs[ld_slot<T>(i)] = i < n4 ? v[j] : f4_zero();
    if (out && i < n4) out[i] = v[j];
  }
}

template <class T, int R, int U>
struct LdTile {
  typename Tile<T>::frag v[R][U];
};
// one row set: base address of row r (wave-uniform), valid 16-byte chunks per row
template <class T, int R, int U>
__device__ __forceinline__ void ld_load(LdTile<T, R, U>& t, const T* const (&row)[R], int b0, int nblk, int nch, int lane) {
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int b = b0 + u;
    if (b < nblk) {  // uniform
      int c = b * 64 + lane;
      c = c < nch ? c : nch - 1;
#pragma unroll
      for (int r = 0; r < R; ++r) t.v[r][u] = ld_nt((const typename Tile<T>::frag*)row[r] + c);
    }
  }
}
template <class T>
__device__ __forceinline__ float ld_dot(const typename Tile<T>::frag& w, const f32x4* x /* plane stride 64 */, float acc) {
#pragma unroll
  for (int p = 0; p < Ld<T>::P; ++p) {
    const f32x4 v = x[p * 64];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc = __builtin_fmaf((float)w[4 * p + i], v[i], acc);
  }
  return acc;
}
// xs: LDS vectors, xstride floats apart; b0: the tile's first block
template <class T, int R, int U, int B>
__device__ __forceinline__ void ld_fma(const LdTile<T, R, U>& t, const float* xs, int xstride, int b0, int nblk, int lane,
                                       float (&acc)[R][B]) {
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int b = b0 + u;
    if (b < nblk) {
#pragma unroll
      for (int q = 0; q < B; ++q) {
        const f32x4* x = (const f32x4*)(xs + (size_t)q * xstride + (size_t)b * Ld<T>::BE) + lane;
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r][q] = ld_dot<T>(t.v[r][u], x, acc[r][q]);
      }
    }
  }
}
// the rest of a row set behind its first tile
template <class T, int R, int U, int B>
__device__ __forceinline__ void ld_rows(LdTile<T, R, U>& t, const T* const (&row)[R], int nblk, int nch, const float* xs,
                                        int xstride, int lane, float (&acc)[R][B]) {
  for (int b0 = 0; b0 < nblk; b0 += U) {
    if (b0) ld_load<T, R, U>(t, row, b0, nblk, nch, lane);
    ld_fma<T, R, U, B>(t, xs, xstride, b0, nblk, lane, acc);
  }
}
template <int R, int B>
__device__ __forceinline__ void ld_reduce(float (&acc)[R][B]) {
#pragma unroll
  for (int r = 0; r < R; ++r)
#pragma unroll
    for (int q = 0; q < B; ++q) acc[r][q] = wave_sum(acc[r][q]);
}
// value (r, q) picked by a lane-dependent index without dynamic register indexing
template <int R, int B>
__device__ __forceinline__ float ld_pick(const float (&acc)[R][B], int r, int q) {
  float v = 0.f;
#pragma unroll
  for (int i = 0; i < R; ++i)
#pragma unroll
    for (int j = 0; j < B; ++j) v = (i == r && j == q) ? acc[i][j] : v;
  return v;
}

struct LdTabs {
  const int32_t *tok, *pos, *slot;  // [B]
};

// The embedding output of a token: scale * embed[token] + pos_emb[position] (pos_emb nullptr: none), rows of ld elements
struct LdEmbed {
  const void *embed, *pos_emb;
  float scale;
};
template <class T>
__device__ __forceinline__ f32x4 ld_embed(const LdEmbed& e, int tok, int pos, int ld, int i4) {
  f32x4 v = quad_f((const T*)e.embed + (size_t)tok * ld + 4 * i4) * e.scale;
  if (e.pos_emb) v += quad_f((const T*)e.pos_emb + (size_t)pos * ld + 4 * i4);
  return v;
}

// ---- k_ld_in -----------------------------------------------------------------------------------------------------
enum LdInKind { LDI_PLAIN = 0, LDI_CONV = 1, LDI_GATED = 2 };
struct LdInSeg {
  const void* w;
  float* out;      // [B][ldo]
  const float* bias;  // LDI_PLAIN: one per row, or nullptr
  int rows, ldo, kind, norm2;  // rows: weight rows (GATED: output columns); norm2: input is the second norm
  int wg0, nwg;
};
struct LdInArgs {
  LdInSeg seg[3];
  int nseg;
  const float* x_in;   // [B][ld]
  float* x_cur;        // written by workgroup 0 when the input is modified
  LdEmbed emb;
  const float* step;
  const float *w1, *b1, *w2, *b2;  // b: nullptr with rms
  float* xn2;          // [B][ld], written by the router's first workgroup (nullptr: nobody reads it)
  int W, ld, from_embed, add_x0, rms;
  float eps;
  GateAct act;
  LdTabs t;
  // LDI_CONV
  const float *conv_w, *conv_b;
  float *conv_st, *xc;  // state + slot * slot_stride ; convolved inputs [B][xc_ld]
  size_t slot_stride;
  int inner, taps, xc_ld;
};

template <class T, int B, int NV>
__global__ __launch_bounds__(256) void k_ld_in(const LdInArgs a) {
  constexpr int R = 4, U = 4;
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  float* xs = (float*)smem_raw;
  __shared__ float red[2 * KH_WAVES_MAX];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, wg = blockIdx.x;
  int si = 0;
  if (a.nseg > 1 && wg >= a.seg[1].wg0) si = 1;
  if (a.nseg > 2 && wg >= a.seg[2].wg0) si = 2;
  // values, not references: a selected address of a kernel argument would force the arguments into scratch memory
  const T* w = (const T*)(si == 0 ? a.seg[0].w : si == 1 ? a.seg[1].w : a.seg[2].w);
  float* out = si == 0 ? a.seg[0].out : si == 1 ? a.seg[1].out : a.seg[2].out;
  const int rows = si == 0 ? a.seg[0].rows : si == 1 ? a.seg[1].rows : a.seg[2].rows;
  const int ldo = si == 0 ? a.seg[0].ldo : si == 1 ? a.seg[1].ldo : a.seg[2].ldo;
  const int kind = si == 0 ? a.seg[0].kind : si == 1 ? a.seg[1].kind : a.seg[2].kind;
  const int norm2 = si == 0 ? a.seg[0].norm2 : si == 1 ? a.seg[1].norm2 : a.seg[2].norm2;
  const int wg0 = si == 0 ? a.seg[0].wg0 : si == 1 ? a.seg[1].wg0 : a.seg[2].wg0;
  const int nwg = si == 0 ? a.seg[0].nwg : si == 1 ? a.seg[1].nwg : a.seg[2].nwg;
  const float* bias = si == 0 ? a.seg[0].bias : si == 1 ? a.seg[1].bias : a.seg[2].bias;
  const int nblk = Ld<T>::blocks(a.ld), nch = a.ld / Ld<T>::E;
  const int per = kind == LDI_GATED ? R / 2 : R;  // outputs per item
  const int items = (rows + per - 1) / per;
  int item = (wg - wg0) * 4 + wave;
  const T* row[R];
  auto set_rows = [&](int it) __attribute__((always_inline)) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      int i;
      if (kind == LDI_GATED) {
        int j = it * 2 + (r & 1);
        j = j < rows ? j : rows - 1;
        i = (j >> 4) * 32 + (j & 15) + (r >> 1) * 16;
      } else {
        i = it * R + r;
        i = i < rows ? i : rows - 1;
      }
      row[r] = w + (size_t)i * a.ld;
    }
  };
  LdTile<T, R, U> t;
  if (item < items) {
    set_rows(item);
    ld_load<T, R, U>(t, row, 0, nblk, nch, lane);
  }
  // convolution operands of the wave's first item: requested with its weights (up to four taps)
  constexpr int CT = 4;
  float cw[CT], cs[CT];
  float cb = 0.f;
  const bool conv_pre = kind == LDI_CONV && a.taps <= CT;
  if (conv_pre && item < items && lane < R * B) {
    const int c = item * R + (lane & (R - 1)), q = lane / R;
    if (c < a.inner) {
      const float* st = a.conv_st + (size_t)a.t.slot[q] * a.slot_stride + c;
      const bool fresh = a.t.pos[q] == 0;
      cb = a.conv_b[c];
#pragma unroll
      for (int k = 0; k < CT; ++k) {
        cw[k] = k < a.taps ? a.conv_w[(size_t)c * a.taps + k] : 0.f;
        cs[k] = k + 1 < a.taps && !fresh ? st[(size_t)k * a.inner] : 0.f;
      }
    }
  }
  const int first_item = item;
  // ---- layer norm of B rows
  const int xstride = nblk * Ld<T>::BE, n4 = a.ld >> 2, total4 = xstride >> 2;
  {
    f32x4 nw[NV], nb[NV], v[NV];
    const f32x4 *wp = (const f32x4*)(norm2 ? a.w2 : a.w1), *bp = (const f32x4*)(norm2 ? a.b2 : a.b1);
    auto get = [&](int q) __attribute__((always_inline)) {
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const int i = threadIdx.x + 256 * j;
        v[j] = f4_zero();
        if (i < n4) {
          v[j] = a.from_embed ? ld_embed<T>(a.emb, a.t.tok[q], a.t.pos[q], a.ld, i) : ((const f32x4*)(a.x_in + (size_t)q * a.ld))[i];
          if (a.add_x0) v[j] += ld_embed<T>(a.emb, a.t.tok[q], a.t.pos[q], a.ld, i);
          if (a.step) v[j] += ((const f32x4*)a.step)[i];
        }
      }
    };
    get(0);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int i = threadIdx.x + 256 * j;
      nw[j] = i < n4 ? wp[i] : f4_zero();
      nb[j] = bp && i < n4 ? bp[i] : f4_zero();
    }
    for (int q = 0; q < B; ++q) {
      if (q) get(q);
      if (a.x_cur && wg == 0) {
#pragma unroll
        for (int j = 0; j < NV; ++j)
          if ((int)threadIdx.x + 256 * j < n4) ((f32x4*)(a.x_cur + (size_t)q * a.ld))[threadIdx.x + 256 * j] = v[j];
      }
      // the router's first workgroup leaves the second norm for the launches that follow
      f32x4* keep = a.xn2 && wg == a.seg[1].wg0 ? (f32x4*)(a.xn2 + (size_t)q * a.ld) : nullptr;
      float shift = 0.f;
      if (!a.rms) shift = a.from_embed ? (float)((const T*)a.emb.embed)[(size_t)a.t.tok[q] * a.ld] : a.x_in[(size_t)q * a.ld];
      if (q) __syncthreads();  // red is free again
      ld_norm<T, NV>(v, nw, nb, shift, a.rms, a.W, n4, total4, a.eps, red, (f32x4*)(xs + (size_t)q * xstride), keep);
    }
  }
  __syncthreads();
  while (item < items) {
    float acc[R][B] = {};
    float bi = 0.f;
    if (bias && lane < R * B) {
      const int i = item * R + (lane & (R - 1));
      bi = bias[i < rows ? i : rows - 1];
    }
    ld_rows<T, R, U, B>(t, row, nblk, nch, xs, xstride, lane, acc);
    const int cur = item;
    item += nwg * 4;
    if (item < items) {  // the next row set travels while this one is reduced
      set_rows(item);
      ld_load<T, R, U>(t, row, 0, nblk, nch, lane);
    }
    ld_reduce<R, B>(acc);
    if (lane < R * B) {
      const int r = lane & (R - 1), q = lane / R;
      if (kind == LDI_GATED) {
        const int j = cur * 2 + r;
        if (r < 2 && j < rows) {
          const float g = ld_pick<R, B>(acc, r, q), u = ld_pick<R, B>(acc, r + 2, q);
          out[(size_t)q * ldo + j] = gated1(a.act, g, u);
        }
      } else {
        const int i = cur * R + r;
        const float v = ld_pick<R, B>(acc, r, q);
        if (i < rows) {
          if (kind == LDI_CONV && i < a.inner) {
            float* st = a.conv_st + (size_t)a.t.slot[q] * a.slot_stride + i;
            float c;
            if (conv_pre && cur == first_item) {
              c = cb;
#pragma unroll
              for (int k = 0; k < CT; ++k) {
                if (k + 1 < a.taps) {
                  c = __builtin_fmaf(cw[k], cs[k], c);
                  if (k) st[(size_t)(k - 1) * a.inner] = cs[k];
                } else if (k + 1 == a.taps) {
                  c = __builtin_fmaf(cw[k], v, c);
                }
              }
            } else {
              const bool fresh = a.t.pos[q] == 0;
              const float* w1 = a.conv_w + (size_t)i * a.taps;
              c = a.conv_b[i];
              for (int k = 0; k + 1 < a.taps; ++k) {
                const float in = fresh ? 0.f : st[(size_t)k * a.inner];
                c = __builtin_fmaf(w1[k], in, c);
                if (k) st[(size_t)(k - 1) * a.inner] = in;
              }
              c = __builtin_fmaf(w1[a.taps - 1], v, c);
            }
            if (a.taps > 1) st[(size_t)(a.taps - 2) * a.inner] = v;
            a.xc[(size_t)q * a.xc_ld + i] = silu1(c);
          } else {
            out[(size_t)q * ldo + i] = v + bi;
          }
        }
      }
    }
  }
}

// ---- k_ld_mid ----------------------------------------------------------------------------------------------------
struct LdMidArgs {
  // experts: workgroups [0, B top nwg_e)
  const float* z;        // [B][ldz]
  const float *corr, *xn2;
  const void* gu;        // experts [2 ffp][ldw]
  float* he;             // [B][top][ffp], weighted
  int32_t* ids;          // [B][top] (-1: identity), written for k_ld_out
  float *id_w, *sh_g;    // [B]
  int nwg_e, top, n_out, n_expert, shared, ffp, ldz, W, ldw, over_chosen;
  GateAct act;
  // mixer: workgroups [.., + nwg_m)
  const void* wm;        // rows x ld
  const float* v;        // [B][ldv] input vectors (n valid entries)
  const float* vnorm;    // RMS norm weight (nullptr: none)
  float* om;             // [B][ldo]
  int nwg_m, rows, ldm, n, n4, ldv, ldo;  // n4: float4 of a row that may be read (no norm)
  // cache rows: the last workgroups (latent attention: one per sequence; heads: one wave per key / value head)
  int latent, heads;
  HeadRow hr;
  const float* raw;      // [B][ldv]: q latent, kv latent, rotated part
  const float* kvn;
  const float2* rope;
  void* cache;
  size_t slot_elems;
  int qr, R, dr, Rp, row, dims;
  float eps;
  LdTabs t;
};
template <class T, int B, int NV, int RP>
__global__ __launch_bounds__(256) void k_ld_mid(const LdMidArgs a) {
  constexpr int R = 4, U = 4;
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  float* xs = (float*)smem_raw;
  __shared__ float red[KH_WAVES_MAX];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  int wg = blockIdx.x;
  LdTile<T, R, U> t;
  const T* row[R];
  const int ne = B * a.top * a.nwg_e;
  if (wg < ne) {  // ---- one chosen expert of one sequence
    const int pair = wg / a.nwg_e, part = wg - pair * a.nwg_e, q = pair / a.top, k = pair - q * a.top;
    const int nblk = Ld<T>::blocks(a.ldw), nch = a.ldw / Ld<T>::E;
    const int n4 = a.ldw >> 2, total4 = nblk * Ld<T>::BE / 4;
    f32x4 x[NV];  // requested first: in flight while the choice is made
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int i = threadIdx.x + 256 * j;
      x[j] = i < n4 ? ((const f32x4*)(a.xn2 + (size_t)q * a.ldw))[i] : f4_zero();
    }
    // every wave makes the choice for itself: its weight loads leave without a barrier
    float idw = 0.f, w = 0.f;
    int id = -1;
    const float wf = moe_route<RP>(a.z + (size_t)q * a.ldz, a.corr, a.n_out, a.top, a.over_chosen, lane,
                                   [&](int kk, int i, float wt) __attribute__((always_inline)) {
      const bool ident = i >= a.n_expert;
      if (ident) idw += wt;
      if (kk == k) {
        id = ident ? -1 : i;
        w = wt;
      }
    });
    w *= wf;
    idw *= wf;
    if (part == 0 && threadIdx.x == 0) {
      a.ids[q * a.top + k] = id;
      if (k == 0) {
        a.id_w[q] = idw;
        if (a.shared) a.sh_g[q] = sigmoid1(a.z[(size_t)q * a.ldz + a.n_out]);
      }
    }
    if (id < 0) return;  // identity expert: no tensors (the whole workgroup agrees)
    const T* base = (const T*)a.gu + (size_t)id * 2 * a.ffp * a.ldw;
    const int items = a.ffp / 2;
    int it = part * 4 + wave;
    auto set_rows = [&](int i) __attribute__((always_inline)) {
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const int j = i * 2 + (r & 1);
        row[r] = base + (size_t)((j >> 4) * 32 + (j & 15) + (r >> 1) * 16) * a.ldw;
      }
    };
    if (it < items) {
      set_rows(it);
      ld_load<T, R, U>(t, row, 0, nblk, nch, lane);
    }
#pragma unroll
    for (int j = 0; j < NV; ++j)
      if ((int)threadIdx.x + 256 * j < total4) ((f32x4*)xs)[ld_slot<T>(threadIdx.x + 256 * j)] = x[j];
    __syncthreads();
    while (it < items) {
      float acc[R][1] = {};
      ld_rows<T, R, U, 1>(t, row, nblk, nch, xs, 0, lane, acc);
      const int cur = it;
      it += a.nwg_e * 4;
      if (it < items) {
        set_rows(it);
        ld_load<T, R, U>(t, row, 0, nblk, nch, lane);
      }
      ld_reduce<R, 1>(acc);
      if (lane < 2) {
        const float g = ld_pick<R, 1>(acc, lane, 0), u = ld_pick<R, 1>(acc, lane + 2, 0);
        a.he[(size_t)pair * a.ffp + cur * 2 + lane] = w * gated1(a.act, g, u);
      }
    }
    return;
  }
  wg -= ne;
  if (wg < a.nwg_m) {  // ---- the mixer's second projection
    const int nblk = Ld<T>::blocks(a.ldm), nch = a.ldm / Ld<T>::E, xstride = nblk * Ld<T>::BE;
    const int items = (a.rows + R - 1) / R;
    int item = wg * 4 + wave;
    auto set_rows = [&](int it) __attribute__((always_inline)) {
#pragma unroll
      for (int r = 0; r < R; ++r) {
        int i = it * R + r;
        i = i < a.rows ? i : a.rows - 1;
        row[r] = (const T*)a.wm + (size_t)i * a.ldm;
      }
    };
    if (item < items) {
      set_rows(item);
      ld_load<T, R, U>(t, row, 0, nblk, nch, lane);
    }
    for (int q = 0; q < B; ++q) {
      const float* v = a.v + (size_t)q * a.ldv;
      f32x4* x4 = (f32x4*)(xs + (size_t)q * xstride);
      if (!a.vnorm) {
        ld_stage<T, 256>(x4, v, a.n4, xstride >> 2, 1.f, threadIdx.x);
      } else {
        float s = 0.f;
        for (int i = threadIdx.x; i < a.n; i += 256) s = __builtin_fmaf(v[i], v[i], s);
        const float rs = 1.0f / sqrtf(block_sum(s, red) / (float)a.n + a.eps);
        for (int i = threadIdx.x; i < xstride; i += 256)
          xs[(size_t)q * xstride + Ld<T>::place(i)] = i < a.n ? v[i] * rs * a.vnorm[i] : 0.f;
      }
    }
    __syncthreads();
    while (item < items) {
      float acc[R][B] = {};
      ld_rows<T, R, U, B>(t, row, nblk, nch, xs, xstride, lane, acc);
      const int cur = item;
      item += a.nwg_m * 4;
      if (item < items) {
        set_rows(item);
        ld_load<T, R, U>(t, row, 0, nblk, nch, lane);
      }
      ld_reduce<R, B>(acc);
      if (lane < R * B) {
        const int r = lane & (R - 1), q = lane / R, i = cur * R + r;
        const float v = ld_pick<R, B>(acc, r, q);
        if (i < a.rows) a.om[(size_t)q * a.ldo + i] = v;
      }
    }
    return;
  }
  wg -= a.nwg_m;
  if (a.heads) {
    const int i = wg * 4 + wave, q = i / a.hr.G, g = i - q * a.hr.G;
    if (q < B)
      heads_cache_row(a.hr, a.raw + (size_t)q * a.ldv, (T*)a.cache + (size_t)a.t.slot[q] * a.slot_elems, a.t.pos[q], g, lane);
    return;
  }
  if (!a.latent || wg >= B) return;  // ---- cache row of sequence wg
  const float* rr = a.raw + (size_t)wg * a.ldv + a.qr;
  const int pos = a.t.pos[wg];
  float s = 0.f;
  for (int i = threadIdx.x; i < a.R; i += 256) s = __builtin_fmaf(rr[i], rr[i], s);
  const float rk = 1.0f / sqrtf(block_sum(s, red) / (float)a.R + a.eps);
  T* crow = (T*)a.cache + (size_t)a.t.slot[wg] * a.slot_elems + (size_t)pos * a.row;
  for (int i = threadIdx.x; i < a.row; i += 256) {
    float v = 0.f;
    if (i < a.R) {
      v = rr[i] * rk * a.kvn[i];
    } else if (i >= a.Rp && i - a.Rp < a.dr) {
      const int j = i - a.Rp;
      v = rr[a.R + j];
      if (j < a.dims) {
        const float2 cs = a.rope[(size_t)pos * (a.dims >> 1) + (j >> 1)];
        const float o = rr[a.R + (j ^ 1)];
        v = (j & 1) ? v * cs.x + o * cs.y : v * cs.x - o * cs.y;
      }
    }
    crow[i] = (T)v;
  }
}

// ---- k_ld_scan: 16 lanes per channel, 16 channels per workgroup.  grid (channels / 16, B) ----------------------------
struct LdScanArgs {
  const float *xc, *xz, *dbc;  // [B][xc_ld], [B][2 C] (z half), [B][rankp + 2 N]
  const void* wdt;             // [C][rankp]
  const float *dt_b, *A2, *D;
  float* state;
  float* y;                    // [B][y_ld]
  size_t slot_stride;
  int C, N, rankp, xc_ld, y_ld;
  LdTabs t;
};
template <class T, int NSL /* states per lane */>
__global__ __launch_bounds__(256) void k_ld_scan(const LdScanArgs a) {
  constexpr int E = Tile<T>::N;
  const int q = blockIdx.y, g = threadIdx.x & 15;
  const int c = blockIdx.x * 16 + ((int)threadIdx.x >> 4);
  const bool live = c < a.C;
  const int cc = live ? c : a.C - 1;
  const float* dbc = a.dbc + (size_t)q * (a.rankp + 2 * a.N);
  float* st = a.state + (size_t)a.t.slot[q] * a.slot_stride + (size_t)cc * a.N;
  const bool fresh = a.t.pos[q] == 0;
  float A2[NSL], S[NSL], Bn[NSL], Cn[NSL];
#pragma unroll
  for (int j = 0; j < NSL; ++j) {  // neighbouring lanes own neighbouring states
    const int n = j * 16 + g;
    const bool in = n < a.N;
    A2[j] = in ? a.A2[(size_t)cc * a.N + n] : 0.f;
    S[j] = in && !fresh ? st[n] : 0.f;
    Bn[j] = in ? dbc[a.rankp + n] : 0.f;
    Cn[j] = in ? dbc[a.rankp + a.N + n] : 0.f;
  }
  const float x = a.xc[(size_t)q * a.xc_ld + cc], z = a.xz[(size_t)q * 2 * a.C + a.C + cc];
  float s = 0.f;
  for (int k = g * E; k < a.rankp; k += 16 * E) {
    const typename Tile<T>::frag w = *(const typename Tile<T>::frag*)((const T*)a.wdt + (size_t)cc * a.rankp + k);
#pragma unroll
    for (int e = 0; e < E; ++e) s = __builtin_fmaf((float)w[e], dbc[k + e], s);
  }
  const float dt = softplus1(group_sum<16>(s) + a.dt_b[cc]), dx = dt * x;
  float y = 0.f;
#pragma unroll
  for (int j = 0; j < NSL; ++j) {
    const int n = j * 16 + g;
    S[j] = __builtin_fmaf(__builtin_amdgcn_exp2f(dt * A2[j]), S[j], dx * Bn[j]);
    y = __builtin_fmaf(S[j], Cn[j], y);
    if (live && n < a.N) st[n] = S[j];
  }
  y = group_sum<16>(y);
  if (g == 0 && live) a.y[(size_t)q * a.y_ld + c] = __builtin_fmaf(a.D[c], x, y) * silu1(z);
}

// ---- k_ld_absorb: Q row of every head: W_uk^T q_n and the rotated part.  grid (H nwg, B) ------------------------------
struct LdAbsorbArgs {
  const float* q;     // [B][H (dnp + drp)]
  const void* ukT;    // [H][Rp][dnp]
  const float2* rope;
  void* Q;            // T [B][H][row]
  int H, nwg, dnp, dr, drp, Rp, row, dims;
  LdTabs t;
};
template <class T>
__global__ __launch_bounds__(256) void k_ld_absorb(const LdAbsorbArgs a) {
  constexpr int E = Tile<T>::N;
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  float* v = (float*)smem_raw;  // [dnp]
  const int b = blockIdx.y, h = (int)blockIdx.x / a.nwg, part = (int)blockIdx.x - h * a.nwg;
  const float* q = a.q + ((size_t)b * a.H + h) * (a.dnp + a.drp);
  for (int i = threadIdx.x; i < a.dnp; i += 256) v[i] = q[i];
  T* Q = (T*)a.Q + ((size_t)b * a.H + h) * a.row;
  if (part == 0) {
    const int pos = a.t.pos[b];
    for (int j = threadIdx.x; j < a.drp; j += 256) {
      float r = j < a.dr ? q[a.dnp + j] : 0.f;
      if (j < a.dims) {
        const float2 cs = a.rope[(size_t)pos * (a.dims >> 1) + (j >> 1)];
        const float o = q[a.dnp + (j ^ 1)];
        r = (j & 1) ? r * cs.x + o * cs.y : r * cs.x - o * cs.y;
      }
      Q[a.Rp + j] = (T)r;
    }
  }
  __syncthreads();
  // eight lanes per row
  for (int i = part * 32 + ((int)threadIdx.x >> 3); i < a.Rp; i += a.nwg * 32) {
    const T* w = (const T*)a.ukT + ((size_t)h * a.Rp + i) * a.dnp;
    float s = 0.f;
    for (int k = (threadIdx.x & 7) * E; k < a.dnp; k += 8 * E) {
      const typename Tile<T>::frag f = *(const typename Tile<T>::frag*)(w + k);
#pragma unroll
      for (int e = 0; e < E; ++e) s = __builtin_fmaf((float)f[e], v[k + e], s);
    }
    s = group_sum<8>(s);
    if ((threadIdx.x & 7) == 0) Q[i] = (T)s;
  }
}

// Merge of the time splits of one head: p [splits][C + 4] (C columns, running maximum, sum); its ns filled splits meet in
// sum [256 / (C / 4) groups][C / 4], summed over the groups by the caller.  Returns 1 / sum of the weights and, in grp, the
// number of groups.  fac: one factor per split, ns <= 256
__device__ __forceinline__ float ld_merge_splits(const float* p, int ns, int C, float* fac, float* red, f32x4* sum, int& grp) {
  float m = -INFINITY;
  for (int s = threadIdx.x; s < ns; s += 256) m = fmaxf(m, p[(size_t)s * (C + 4) + C]);
  m = block_max(m, red);
  float l = 0.f;
  for (int s = threadIdx.x; s < ns; s += 256) {
    const float* ps = p + (size_t)s * (C + 4) + C;
    const float f = __builtin_amdgcn_exp2f(ps[0] - m);  // an empty split: exp2(-inf) = 0
    fac[s] = f;
    l = __builtin_fmaf(f, ps[1], l);
  }
  l = block_sum(l, red);
  // column groups of four; 256 / (C / 4) thread groups share the splits and meet in LDS
  const int c4 = C >> 2, g = (int)threadIdx.x / c4;
  grp = c4 < 256 ? 256 / c4 : 1;
  if (g < grp) {
    for (int i = (int)threadIdx.x - g * c4; i < c4; i += 256) {
      f32x4 v = f4_zero();
      int s = g;
      for (; s + 7 * grp < ns; s += 8 * grp) {
        f32x4 x[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) x[j] = *(const f32x4*)(p + (size_t)(s + j * grp) * (C + 4) + 4 * i);
#pragma unroll
        for (int j = 0; j < 8; ++j) v = fma_s(fac[s + j * grp], x[j], v);
      }
      for (; s < ns; s += grp) v = fma_s(fac[s], *(const f32x4*)(p + (size_t)s * (C + 4) + 4 * i), v);
      sum[g * c4 + i] = v;
    }
  }
  __syncthreads();
  return 1.0f / l;
}

// ---- k_ld_values: merge of the time splits, then W_uv of the head.  grid (H nwg, B) ----------------------------------
struct LdValuesArgs {
  const float* part;  // [B H][nsplit][Rp + 4]
  const void* uv;     // [H][dvp][Rp]
  float* o;           // [B][H dvp]
  int H, nwg, nsplit, Rp, dvp;
  const int32_t* pos;
};
template <class T>
__global__ __launch_bounds__(256) void k_ld_values(const LdValuesArgs a) {
  constexpr int R = 4, U = 1;
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  float* xs = (float*)smem_raw;
  __shared__ float fac[256];
  __shared__ float red[KH_WAVES_MAX];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int b = blockIdx.y, h = (int)blockIdx.x / a.nwg, part = (int)blockIdx.x - h * a.nwg;
  const float* p = a.part + ((size_t)b * a.H + h) * a.nsplit * (size_t)(a.Rp + 4);
  const int nblk = Ld<T>::blocks(a.Rp), nch = a.Rp / Ld<T>::E;
  const int items = a.dvp / R;
  int item = part * 4 + wave;
  const T* row[R];
  LdTile<T, R, U> t;
  auto set_rows = [&](int it) __attribute__((always_inline)) {
#pragma unroll
    for (int r = 0; r < R; ++r) row[r] = (const T*)a.uv + ((size_t)h * a.dvp + it * R + r) * a.Rp;
  };
  if (item < items) {
    set_rows(item);
    ld_load<T, R, U>(t, row, 0, nblk, nch, lane);
  }
  const int c4 = a.Rp >> 2;
  f32x4* sum = (f32x4*)(xs + (size_t)nblk * Ld<T>::BE);  // [grp][c4]
  int grp;
  const float inv = ld_merge_splits(p, lat_active_splits(a.pos[b] + 1, a.nsplit), a.Rp, fac, red, sum, grp);
  for (int i = threadIdx.x; i < nblk * Ld<T>::BE / 4; i += 256) {
    f32x4 v = f4_zero();
    if (i < c4)
      for (int k = 0; k < grp; ++k) v += sum[k * c4 + i];
    ((f32x4*)xs)[ld_slot<T>(i)] = v * inv;
  }
  __syncthreads();
  while (item < items) {
    float acc[R][1] = {};
    ld_rows<T, R, U, 1>(t, row, nblk, nch, xs, 0, lane, acc);
    const int cur = item;
    item += a.nwg * 4;
    if (item < items) {
      set_rows(item);
      ld_load<T, R, U>(t, row, 0, nblk, nch, lane);
    }
    ld_reduce<R, 1>(acc);
    if (lane < R) a.o[((size_t)b * a.H + h) * a.dvp + cur * R + lane] = ld_pick<R, 1>(acc, lane, 0);
  }
}

// ---- k_ld_merge: attention over heads: merge of the time splits, output gate.  grid (H, B) --------------------------
struct LdMergeArgs {
  const float* part;  // [B H][nsplit][C + 4]
  const float* gate;  // [B][ldg]: logits head by head, gs apart (nullptr: none)
  float* o;           // [B][ldo], heads gs apart
  int H, nsplit, C, gs, ldg, ldo;
  KeySpan span;
  const int32_t* pos;
};
static __global__ __launch_bounds__(256) void k_ld_merge(const LdMergeArgs a) {
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  f32x4* sum = (f32x4*)smem_raw;
  __shared__ float fac[256];
  __shared__ float red[KH_WAVES_MAX];
  const int b = blockIdx.y, h = blockIdx.x, pos = a.pos[b], i = (int)threadIdx.x, c4 = a.C >> 2;
  f32x4 g = f4_zero();
  const bool live = 4 * i < a.gs;
  if (a.gate && live) g = *(const f32x4*)(a.gate + (size_t)b * a.ldg + (size_t)h * a.gs + 4 * i);
  int grp;
  const float inv = ld_merge_splits(a.part + ((size_t)b * a.H + h) * a.nsplit * (size_t)(a.C + 4),
                                    lat_active_splits(pos + 1 - a.span.first(pos), a.nsplit), a.C, fac, red, sum, grp);
  if (!live) return;
  f32x4 v = f4_zero();
  for (int k = 0; k < grp; ++k) v += sum[k * c4 + i];
#pragma unroll
  for (int j = 0; j < 4; ++j) v[j] *= a.gate ? inv * sigmoid1(g[j]) : inv;
  *(f32x4*)(a.o + (size_t)b * a.ldo + (size_t)h * a.gs + 4 * i) = v;
}

// ---- k_ld_enter: x_out = W [x ; embedding output], a pass of a loop that enters through a matrix --------------------
struct LdEnterArgs {
  const void* w;      // [W][2 ld]
  const float* x;     // [B][ld] (nullptr: the embedding output itself)
  float* x_out;       // [B][ld]
  LdEmbed emb;
  int W, ld, ks;
  LdTabs t;
};
// Workgroup = 8 waves = 8 / ks groups of ks waves; a group owns R rows, its waves share the blocks.
template <class T, int B>
__global__ __launch_bounds__(512) void k_ld_enter(const LdEnterArgs a) {
  constexpr int R = 2, U = 4, BE = Ld<T>::BE;
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  float* xs = (float*)smem_raw;
  __shared__ float comb[8][R * B];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int K = 2 * a.ld, nblk = Ld<T>::blocks(K), nch = K / Ld<T>::E, n4 = a.ld >> 2;
  const int kp = wave % a.ks, item = ((int)blockIdx.x * (8 / a.ks) + wave / a.ks) * R;
  const int per = (nblk + a.ks - 1) / a.ks, b0 = kp * per, b1 = b0 + per < nblk ? b0 + per : nblk;
  const T* row[R];
#pragma unroll
  for (int r = 0; r < R; ++r) row[r] = (const T*)a.w + (size_t)(item + r < a.W ? item + r : a.W - 1) * K;
  LdTile<T, R, U> t;
  ld_load<T, R, U>(t, row, b0, b1, nch, lane);
  for (int q = 0; q < B; ++q) {
    f32x4* xq = (f32x4*)(xs + (size_t)q * nblk * BE);
    for (int i = threadIdx.x; i < nblk * BE / 4; i += 512) {
      f32x4 v = f4_zero();
      if (i < n4 && a.x) v = ((const f32x4*)(a.x + (size_t)q * a.ld))[i];
      else if (i < 2 * n4) v = ld_embed<T>(a.emb, a.t.tok[q], a.t.pos[q], a.ld, i < n4 ? i : i - n4);
      xq[ld_slot<T>(i)] = v;
    }
  }
  __syncthreads();
  float acc[R][B] = {};
  for (int b = b0; b < b1; b += U) {
    if (b != b0) ld_load<T, R, U>(t, row, b, b1, nch, lane);
    ld_fma<T, R, U, B>(t, xs, nblk * BE, b, b1, lane, acc);
  }
  ld_reduce<R, B>(acc);
  if (lane < R * B) comb[wave][lane] = ld_pick<R, B>(acc, lane & (R - 1), lane / R);
  __syncthreads();
  if (kp == 0 && lane < R * B) {
    float v = 0.f;
    for (int k = 0; k < a.ks; ++k) v += comb[wave + k][lane];
    const int q = lane / R, i = item + (lane & (R - 1));
    if (i < a.W) a.x_out[(size_t)q * a.ld + i] = v;
  }
}

// ---- k_ld_out ----------------------------------------------------------------------------------------------------
struct LdOutArgs {
  const void* wo;         // [W][ldv]
  const float* v;         // [B][ld_v] mixer vector (4 n4v readable)
  const void *down, *sdown;  // experts [W][ffp] each; shared [W][sffp]
  const float *he, *hs;   // [B][top][ffp] (weighted), [B][sffp]
  const int32_t* ids;     // [B][top]
  const float *id_w, *sh_g, *xn2, *x_cur;  // id_w, sh_g: nullptr = none, 1
  const float* bias;      // of W_o, or nullptr
  float* x_out;           // [B][ld]
  int W, ld, n4v, ld_v, ldv, top, ffp, sffp, moe, ks;
  float mult;             // of everything that is added to the residual
};
// Workgroup = 8 waves = 8 / ks groups of ks waves; a group owns R rows, its waves share the blocks of the concatenation
// [mixer | shared | expert 0 | expert 1 ...] (blocks of identity experts are skipped).  Experts differ between
// sequences, so for B > 1 the feed-forward part runs once per sequence.  A block's place follows from its number, so
// the first two tiles of a wave are requested before the vectors are staged.
template <class T, int B>
__global__ __launch_bounds__(512) void k_ld_out(const LdOutArgs a) {
  constexpr int R = 2, U = 4;
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  typedef typename Tile<T>::frag frag;
  constexpr int BE = Ld<T>::BE, E = Ld<T>::E;
  __shared__ float comb[8][R * B];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int nbv = Ld<T>::blocks(a.ldv);
  const int nbe = a.moe && a.top ? Ld<T>::blocks(a.ffp) : 1, nbs = a.moe && a.sffp ? Ld<T>::blocks(a.sffp) : 0;
  const int nb = nbv + nbs + (a.moe ? a.top * nbe : 0);
  float* xv = (float*)smem_raw;
  float* xf = xv + (size_t)B * nbv * BE;
  const int kp = wave % a.ks, grp = (int)blockIdx.x * (8 / a.ks) + wave / a.ks;
  const int item = grp * R;
  int ri[R];
#pragma unroll
  for (int r = 0; r < R; ++r) ri[r] = item + r < a.W ? item + r : a.W - 1;
  // residual operands of the rows this wave will finish
  float rx = 0.f, rn = 0.f, rw = 0.f, rb = 0.f;
  if (kp == 0 && lane < R * B) {
    const int q = lane / R, i = item + (lane & (R - 1));
    if (i < a.W) {
      rx = a.x_cur[(size_t)q * a.ld + i];
      if (a.bias) rb = a.bias[i];
      if (a.id_w) {
        rn = a.xn2[(size_t)q * a.ld + i];
        rw = a.id_w[q];
      }
    }
  }
  frag w[2][R][U];
  int nc[2][U];
  auto fetch = [&](int set, int b0, int b1, int q) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int b = b0 + u;  // wave-uniform
      nc[set][u] = 0;
      if (b < b1) {
        const T* p = (const T*)a.wo;
        int stride = a.ldv, bb = b;
        bool have = true;
        if (b >= nbv + nbs) {
          const int e = b - nbv - nbs, k = e / nbe, id = a.ids[q * a.top + k];
          bb = e - k * nbe;
          stride = a.ffp;
          have = id >= 0;
          p = (const T*)a.down + (size_t)(have ? id : 0) * a.W * a.ffp;
        } else if (b >= nbv) {
          bb = b - nbv;
          stride = a.sffp;
          p = (const T*)a.sdown;
        }
        const int left = stride / E - bb * 64, n = left < 64 ? left : 64;
        nc[set][u] = have ? n : 0;
        if (have) {
          const int c = lane < n ? lane : n - 1;
#pragma unroll
          for (int r = 0; r < R; ++r) w[set][r][u] = ld_nt((const frag*)(p + (size_t)ri[r] * stride + (size_t)bb * BE) + c);
        }
      }
    }
  };
  float acc[R][B] = {};
#pragma unroll
  for (int q = 0; q < B; ++q) {
    const int b_lo = q == 0 ? 0 : nbv, per = (nb - b_lo + a.ks - 1) / a.ks;
    const int b0 = b_lo + kp * per, b1 = b0 + per < nb ? b0 + per : nb;
    fetch(0, b0, b1, q);
    fetch(1, b0 + U, b1, q);
    if (q == 0) {
      for (int j = 0; j < B; ++j)
        ld_stage<T, 512>((f32x4*)(xv + (size_t)j * nbv * BE), a.v + (size_t)j * a.ld_v, a.n4v, nbv * BE / 4, 1.f, threadIdx.x);
    } else {
      __syncthreads();  // the feed-forward vectors of the sequence before have been consumed
    }
    if (a.moe) {
      if (nbs) ld_stage<T, 512>((f32x4*)xf, a.hs + (size_t)q * a.sffp, a.sffp >> 2, nbs * BE / 4, a.sh_g ? a.sh_g[q] : 1.f,
                                 threadIdx.x);
      for (int k = 0; k < a.top; ++k)
        ld_stage<T, 512>((f32x4*)(xf + (size_t)(nbs + k * nbe) * BE), a.he + (size_t)(q * a.top + k) * a.ffp, a.ffp >> 2,
                         nbe * BE / 4, 1.f, threadIdx.x);
    }
    __syncthreads();
    auto use = [&](int set, int b) __attribute__((always_inline)) {
#pragma unroll
      for (int u = 0; u < U; ++u) {
        if (!nc[set][u]) continue;
        if (b + u < nbv) {
#pragma unroll
          for (int j = 0; j < B; ++j) {
            const f32x4* x = (const f32x4*)(xv + ((size_t)j * nbv + b + u) * BE) + lane;
#pragma unroll
            for (int r = 0; r < R; ++r) acc[r][j] = ld_dot<T>(w[set][r][u], x, acc[r][j]);
          }
        } else {
          const f32x4* x = (const f32x4*)(xf + (size_t)(b + u - nbv) * BE) + lane;
#pragma unroll
          for (int r = 0; r < R; ++r) acc[r][q] = ld_dot<T>(w[set][r][u], x, acc[r][q]);
        }
      }
    };
    for (int b = b0; b < b1; b += 2 * U) {
      use(0, b);
      fetch(0, b + 2 * U, b1, q);
      use(1, b + U);
      fetch(1, b + 3 * U, b1, q);
    }
  }
  ld_reduce<R, B>(acc);
  if (lane < R * B) comb[wave][lane] = ld_pick<R, B>(acc, lane & (R - 1), lane / R);
  __syncthreads();
  if (kp == 0 && lane < R * B) {
    float v = 0.f;
    for (int k = 0; k < a.ks; ++k) v += comb[wave + k][lane];
    const int q = lane / R, i = item + (lane & (R - 1));
    if (i < a.W) a.x_out[(size_t)q * a.ld + i] = __builtin_fmaf(a.mult, __builtin_fmaf(rw, rn, v) + rb, rx);
  }
}

// ---- k_ld_head ---------------------------------------------------------------------------------------------------
struct LdHeadArgs {
  const float* x;        // [B][ld]
  const float *w, *b;    // final norm (rms: b may be nullptr)
  const void* head;      // [V][ld]
  float* logits;         // [B][V]
  float* part_val;       // argmax partials of sequence 0 (nullptr: none)
  int32_t* part_idx;
  int W, ld, V, rms;
  float eps, cap;
};
template <class T, int B, int NV>
__global__ __launch_bounds__(256) void k_ld_head(const LdHeadArgs a) {
  constexpr int R = 4, U = 4;
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  float* xs = (float*)smem_raw;
  __shared__ float red[2 * KH_WAVES_MAX];
  __shared__ float sv[4];
  __shared__ int si[4];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int nblk = Ld<T>::blocks(a.ld), nch = a.ld / Ld<T>::E, xstride = nblk * Ld<T>::BE;
  const int items = (a.V + R - 1) / R;
  int item = blockIdx.x * 4 + wave;
  const T* row[R];
  LdTile<T, R, U> t;
  auto set_rows = [&](int it) __attribute__((always_inline)) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      int i = it * R + r;
      i = i < a.V ? i : a.V - 1;
      row[r] = (const T*)a.head + (size_t)i * a.ld;
    }
  };
  if (item < items) {
    set_rows(item);
    ld_load<T, R, U>(t, row, 0, nblk, nch, lane);
  }
  {
    const int n4 = a.ld >> 2;
    f32x4 nw[NV], nb[NV], v[NV];
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int i = threadIdx.x + 256 * j;
      nw[j] = i < n4 ? ((const f32x4*)a.w)[i] : f4_zero();
      nb[j] = a.b && i < n4 ? ((const f32x4*)a.b)[i] : f4_zero();
    }
    for (int q = 0; q < B; ++q) {
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const int i = threadIdx.x + 256 * j;
        v[j] = i < n4 ? ((const f32x4*)(a.x + (size_t)q * a.ld))[i] : f4_zero();
      }
      if (q) __syncthreads();
      ld_norm<T, NV>(v, nw, nb, a.rms ? 0.f : a.x[(size_t)q * a.ld], a.rms, a.W, n4, xstride >> 2, a.eps, red, (f32x4*)(xs + (size_t)q * xstride), nullptr);
    }
  }
  __syncthreads();
  float bv = -INFINITY;
  int bi = 0x7fffffff;
  while (item < items) {
    float acc[R][B] = {};
    ld_rows<T, R, U, B>(t, row, nblk, nch, xs, xstride, lane, acc);
    const int cur = item;
    item += gridDim.x * 4;
    if (item < items) {
      set_rows(item);
      ld_load<T, R, U>(t, row, 0, nblk, nch, lane);
    }
    ld_reduce<R, B>(acc);
    if (lane < R * B) {
      const int r = lane & (R - 1), q = lane / R, i = cur * R + r;
      float v = ld_pick<R, B>(acc, r, q);
      if (a.cap > 0.f) v = a.cap * tanhf(v / a.cap);
      if (i < a.V) {
        a.logits[(size_t)q * a.V + i] = v;
        if (q == 0) amax_merge(bv, bi, v, i);
      }
    }
  }
  if (a.part_val) {
    wave_amax(bv, bi);
    if (lane == 0) {
      sv[wave] = bv;
      si[wave] = bi;
    }
    __syncthreads();
    if (threadIdx.x == 0) {
#pragma unroll
      for (int w = 1; w < 4; ++w) amax_merge(bv, bi, sv[w], si[w]);
      a.part_val[blockIdx.x] = bv;
      a.part_idx[blockIdx.x] = bi;
    }
  }
}
}  // namespace khm
