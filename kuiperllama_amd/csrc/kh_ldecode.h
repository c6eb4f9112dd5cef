// kh_ldecode.h — fused decode step of the layer-list models: B sequences (1, 2 or 4), one token each.
//
// Per layer   mixer mamba1: 4 launches      latent attention: 6 launches
//   k_ld_in   layer norms -> LDS ; every projection that reads them: mixer input, router (+ shared gate row), shared
//             expert gate / up with SwiGLU ; mamba x rows go through the convolution and silu in the epilogue
//   k_ld_mid  router choice, chosen experts' gate / up ; mamba: W_x ; latent: W_uq behind its RMS norm, cache row
//   mamba     k_ld_scan   dt projection, softplus, one step of the selective scan, gate
//   latent    k_ld_absorb W_uk^T q per head, rotation ; k_latent_attn (time splits) ; k_ld_values merge + W_uv per head
//   k_ld_out  W_o . v + experts' down + shared down + identity experts + residual, one dot product per row over a
//             concatenation of weight rows
// then k_ld_head (final norm, head, soft cap, argmax partials) and the sampler of kh_fused.h.
//
// GEMV core: a wave owns R rows.  A row is cut into BLOCKS of 64 x 16 bytes; U blocks of R rows are requested together
// (non-temporal), and the first tile of a wave is requested before the input vectors are staged.  Vectors lie in LDS
// as fp32, block by block, split into planes of four so that a lane's reads are consecutive 16-byte slots; their tails
// are zeros, so the clamped weight loads of a tail lane contribute nothing.  Accumulation is fp32.
#pragma once
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

// ---- k_ld_in -----------------------------------------------------------------------------------------------------
enum LdInKind { LDI_PLAIN = 0, LDI_CONV = 1, LDI_SWIGLU = 2 };
struct LdInSeg {
  const void* w;
  float* out;      // [B][ldo]
  int rows, ldo, kind, norm2;  // rows: weight rows (SWIGLU: output columns); norm2: input is the second norm
  int wg0, nwg;
};
struct LdInArgs {
  LdInSeg seg[3];
  int nseg;
  const float* x_in;   // [B][W]
  float* x_cur;        // written by workgroup 0 when the input is modified
  const void* embed;
  const float* step;
  const float *w1, *b1, *w2, *b2;
  float* xn2;          // [B][W], written by workgroup 0 (nullptr: no feed-forward)
  int W, ld, from_embed, add_x0;
  float eps;
  LdTabs t;
  // LDI_CONV
  const float *conv_w, *conv_b;
  float *conv_st, *xc;  // state + slot * slot_stride ; convolved inputs [B][xc_ld]
  size_t slot_stride;
  int inner, taps, xc_ld;
};

template <class T, int B>
__global__ __launch_bounds__(256) void k_ld_in(const LdInArgs a) {
  constexpr int R = 4, U = 4;
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  float* xs = (float*)smem_raw;
  __shared__ float red[KH_WAVES_MAX];
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
  const int nblk = Ld<T>::blocks(a.ld), nch = a.ld / Ld<T>::E;
  const int per = kind == LDI_SWIGLU ? R / 2 : R;  // outputs per item
  const int items = (rows + per - 1) / per;
  int item = (wg - wg0) * 4 + wave;
  const T* row[R];
  auto set_rows = [&](int it) __attribute__((always_inline)) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      int i;
      if (kind == LDI_SWIGLU) {
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
  // ---- layer norm of B rows
  const int xstride = nblk * Ld<T>::BE;
  for (int q = 0; q < B; ++q) {
    const int tok = a.t.tok[q];
    const T* e = (const T*)a.embed + (size_t)tok * a.W;
    float* x = xs + (size_t)q * xstride;
    float s = 0.f;
    for (int i = threadIdx.x; i < xstride; i += 256) {
      float v = 0.f;
      if (i < a.W) {
        v = a.from_embed ? (float)e[i] : a.x_in[(size_t)q * a.W + i];
        if (a.add_x0) v += (float)e[i];
        if (a.step) v += a.step[i];
        if (a.x_cur && wg == 0) a.x_cur[(size_t)q * a.W + i] = v;
      }
      x[Ld<T>::place(i)] = v;
      s += v;
    }
    const float mean = block_sum(s, red) / (float)a.W;
    float d2 = 0.f;
    for (int i = threadIdx.x; i < a.W; i += 256) {
      const float d = x[Ld<T>::place(i)] - mean;
      d2 = __builtin_fmaf(d, d, d2);
    }
    const float rstd = 1.0f / sqrtf(block_sum(d2, red) / (float)a.W + a.eps);
    for (int i = threadIdx.x; i < a.W; i += 256) {
      const float n = (x[Ld<T>::place(i)] - mean) * rstd;
      float y1 = 0.f;
      if (norm2) y1 = n * a.w2[i] + a.b2[i];
      else y1 = n * a.w1[i] + a.b1[i];
      x[Ld<T>::place(i)] = y1;
      if (a.xn2 && wg == 0) a.xn2[(size_t)q * a.W + i] = n * a.w2[i] + a.b2[i];
    }
  }
  __syncthreads();
  while (item < items) {
    float acc[R][B] = {};
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
      if (kind == LDI_SWIGLU) {
        const int j = cur * 2 + r;
        if (r < 2 && j < rows) {
          const float g = ld_pick<R, B>(acc, r, q), u = ld_pick<R, B>(acc, r + 2, q);
          out[(size_t)q * ldo + j] = silu1(g) * u;
        }
      } else {
        const int i = cur * R + r;
        const float v = ld_pick<R, B>(acc, r, q);
        if (i < rows) {
          if (kind == LDI_CONV && i < a.inner) {
            float* st = a.conv_st + (size_t)a.t.slot[q] * a.slot_stride + i;
            const bool fresh = a.t.pos[q] == 0;
            const float* cw = a.conv_w + (size_t)i * a.taps;
            float c = a.conv_b[i];
            for (int k = 0; k + 1 < a.taps; ++k) {
              const float in = fresh ? 0.f : st[(size_t)k * a.inner];
              c = __builtin_fmaf(cw[k], in, c);
              if (k) st[(size_t)(k - 1) * a.inner] = in;
            }
            c = __builtin_fmaf(cw[a.taps - 1], v, c);
            if (a.taps > 1) st[(size_t)(a.taps - 2) * a.inner] = v;
            a.xc[(size_t)q * a.xc_ld + i] = silu1(c);
          } else {
            out[(size_t)q * ldo + i] = v;
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
  int nwg_e, top, n_out, n_expert, shared, ffp, ldz, W, ldw;
  // mixer: workgroups [.., + nwg_m)
  const void* wm;        // rows x ld
  const float* v;        // [B][ldv] input vectors (n valid entries)
  const float* vnorm;    // RMS norm weight (nullptr: none)
  float* om;             // [B][ldo]
  int nwg_m, rows, ldm, n, ldv, ldo;
  // cache rows of latent attention: the last B workgroups
  int latent;
  const float* raw;      // [B][ldv]: q latent, kv latent, rotated part
  const float* kvn;
  const float2* rope;
  void* cache;
  size_t slot_elems;
  int qr, R, dr, Rp, row, dims;
  float eps;
  LdTabs t;
};
template <class T, int B>
__global__ __launch_bounds__(256) void k_ld_mid(const LdMidArgs a) {
  constexpr int R = 4, U = 4;
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  float* xs = (float*)smem_raw;
  __shared__ float red[KH_WAVES_MAX];
  __shared__ int s_id;
  __shared__ float s_w;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  int wg = blockIdx.x;
  LdTile<T, R, U> t;
  const T* row[R];
  const int ne = B * a.top * a.nwg_e;
  if (wg < ne) {  // ---- one chosen expert of one sequence
    const int pair = wg / a.nwg_e, part = wg - pair * a.nwg_e, q = pair / a.top, k = pair - q * a.top;
    if (wave == 0) {
      float idw = 0.f;
      moe_route(a.z + (size_t)q * a.ldz, a.corr, a.n_out, a.top, lane, [&](int kk, int id, float w) __attribute__((always_inline)) {
        const bool ident = id >= a.n_expert;
        if (ident) idw += w;
        if (kk == k && lane == 0) {
          s_id = ident ? -1 : id;
          s_w = w;
          if (part == 0) a.ids[q * a.top + k] = ident ? -1 : id;
        }
      });
      if (k == 0 && part == 0 && lane == 0) {
        a.id_w[q] = idw;
        if (a.shared) a.sh_g[q] = sigmoid1(a.z[(size_t)q * a.ldz + a.n_out]);
      }
    }
    const int nblk = Ld<T>::blocks(a.ldw), nch = a.ldw / Ld<T>::E;
    for (int i = threadIdx.x; i < nblk * Ld<T>::BE; i += 256)
      xs[Ld<T>::place(i)] = i < a.W ? a.xn2[(size_t)q * a.W + i] : 0.f;
    __syncthreads();
    const int id = s_id;
    if (id < 0) return;  // identity expert: no tensors
    const float w = s_w;
    const T* base = (const T*)a.gu + (size_t)id * 2 * a.ffp * a.ldw;
    const int items = a.ffp / 2;
    for (int it = part * 4 + wave; it < items; it += a.nwg_e * 4) {
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const int j = it * 2 + (r & 1);
        row[r] = base + (size_t)((j >> 4) * 32 + (j & 15) + (r >> 1) * 16) * a.ldw;
      }
      float acc[R][1] = {};
      ld_load<T, R, U>(t, row, 0, nblk, nch, lane);
      ld_rows<T, R, U, 1>(t, row, nblk, nch, xs, 0, lane, acc);
      ld_reduce<R, 1>(acc);
      if (lane < 2) {
        const float g = ld_pick<R, 1>(acc, lane, 0), u = ld_pick<R, 1>(acc, lane + 2, 0);
        a.he[(size_t)pair * a.ffp + it * 2 + lane] = w * (silu1(g) * u);
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
      float s = 0.f;
      for (int i = threadIdx.x; i < xstride; i += 256) {
        const float v = i < a.n ? a.v[(size_t)q * a.ldv + i] : 0.f;
        xs[(size_t)q * xstride + Ld<T>::place(i)] = v;
        s = __builtin_fmaf(v, v, s);
      }
      if (a.vnorm) {
        const float rs = 1.0f / sqrtf(block_sum(s, red) / (float)a.n + a.eps);
        for (int i = threadIdx.x; i < a.n; i += 256) xs[(size_t)q * xstride + Ld<T>::place(i)] *= rs * a.vnorm[i];
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

// ---- k_ld_scan: grid (channels / (256 / G), B) --------------------------------------------------------------------
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
template <class T, int G>
__global__ __launch_bounds__(256) void k_ld_scan(const LdScanArgs a) {
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  constexpr int CW = 256 / G;           // channels of a workgroup
  constexpr int E = Tile<T>::N;
  float* v = (float*)smem_raw;          // dt inputs [rankp], B [G 8], C [G 8]
  const int NP = G * KH_SCAN_NS;
  float* bc = v + a.rankp;
  float* dts = bc + 2 * NP;             // [CW]
  const int q = blockIdx.y, c0 = blockIdx.x * CW;
  const float* dbc = a.dbc + (size_t)q * (a.rankp + 2 * a.N);
  const int g = threadIdx.x & (G - 1), cl = (int)threadIdx.x / G;
  const int c = c0 + cl;
  const bool live = c < a.C;
  const int cc = live ? c : a.C - 1;
  float* st = a.state + (size_t)a.t.slot[q] * a.slot_stride + (size_t)cc * a.N;
  const bool fresh = a.t.pos[q] == 0;
  float A2[KH_SCAN_NS], S[KH_SCAN_NS];
#pragma unroll
  for (int j = 0; j < KH_SCAN_NS; ++j) {
    const int n = g * KH_SCAN_NS + j;
    A2[j] = n < a.N ? a.A2[(size_t)cc * a.N + n] : 0.f;
    S[j] = n < a.N && !fresh ? st[n] : 0.f;
  }
  for (int i = threadIdx.x; i < a.rankp; i += 256) v[i] = dbc[i];
  for (int i = threadIdx.x; i < 2 * NP; i += 256) {
    const int which = i >= NP, n = i - which * NP;
    bc[i] = n < a.N ? dbc[a.rankp + which * a.N + n] : 0.f;
  }
  __syncthreads();
  // dt: eight lanes per channel
  for (int i = (int)threadIdx.x >> 3; i < CW; i += 32) {
    const int ch = c0 + i < a.C ? c0 + i : a.C - 1;
    float s = 0.f;
    for (int k = (threadIdx.x & 7) * E; k < a.rankp; k += 8 * E) {
      const typename Tile<T>::frag w = *(const typename Tile<T>::frag*)((const T*)a.wdt + (size_t)ch * a.rankp + k);
#pragma unroll
      for (int e = 0; e < E; ++e) s = __builtin_fmaf((float)w[e], v[k + e], s);
    }
    s = group_sum<8>(s);
    if ((threadIdx.x & 7) == 0) dts[i] = softplus1(s + a.dt_b[ch]);
  }
  __syncthreads();
  const float dt = dts[cl], x = a.xc[(size_t)q * a.xc_ld + cc], dx = dt * x;
  float y = 0.f;
#pragma unroll
  for (int j = 0; j < KH_SCAN_NS; ++j) {
    const int n = g * KH_SCAN_NS + j;
    S[j] = __builtin_fmaf(__builtin_amdgcn_exp2f(dt * A2[j]), S[j], dx * bc[n]);
    y = __builtin_fmaf(S[j], bc[NP + n], y);
    if (live && n < a.N) st[n] = S[j];
  }
  y = group_sum<G>(y);
  if (g == 0 && live) {
    y = __builtin_fmaf(a.D[c], x, y);
    a.y[(size_t)q * a.y_ld + c] = y * silu1(a.xz[(size_t)q * 2 * a.C + a.C + c]);
  }
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
  const int ns = lat_active_splits(a.pos[b] + 1, a.nsplit);
  float m = -INFINITY;
  for (int s = threadIdx.x; s < ns; s += 256) m = fmaxf(m, p[(size_t)s * (a.Rp + 4) + a.Rp]);
  m = block_max(m, red);
  float l = 0.f;
  for (int s = threadIdx.x; s < ns; s += 256) {
    const float* ps = p + (size_t)s * (a.Rp + 4) + a.Rp;
    const float f = __builtin_amdgcn_exp2f(ps[0] - m);  // an empty split: exp2(-inf) = 0
    fac[s] = f;
    l = __builtin_fmaf(f, ps[1], l);
  }
  l = block_sum(l, red);
  const float inv = 1.0f / l;
  for (int i = threadIdx.x; i < nblk * Ld<T>::BE; i += 256) {
    float v = 0.f;
    if (i < a.Rp)
      for (int s = 0; s < ns; ++s) v = __builtin_fmaf(fac[s], p[(size_t)s * (a.Rp + 4) + i], v);
    xs[Ld<T>::place(i)] = v * inv;
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

// ---- k_ld_out ----------------------------------------------------------------------------------------------------
struct LdOutArgs {
  const void* wo;         // [W][ldv]
  const float* v;         // [B][ld_v] mixer vector (n_v valid)
  const void *down, *sdown;  // experts [W][ffp] each; shared [W][sffp]
  const float *he, *hs;   // [B][top][ffp] (weighted), [B][sffp]
  const int32_t* ids;     // [B][top]
  const float *id_w, *sh_g, *xn2, *x_cur;
  float* x_out;           // [B][W]
  int W, n_v, ld_v, ldv, top, ffp, sffp, moe, nwg;
};
// A row of the concatenation is a list of blocks: table entry = weight pointer of row 0 at the block, row stride and
// valid chunks.  Vector parts lie block by block in the same order.
struct LdBlk {
  const void* p;
  int stride, nch;  // elements between rows; 16-byte chunks valid in this block
};
template <class T, int B>
__global__ __launch_bounds__(256) void k_ld_out(const LdOutArgs a) {
  constexpr int R = 2, U = 8;
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  typedef typename Tile<T>::frag frag;
  constexpr int BE = Ld<T>::BE, E = Ld<T>::E;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int nbv = Ld<T>::blocks(a.ldv);
  const int nbe = a.moe ? Ld<T>::blocks(a.ffp) : 0, nbs = a.moe && a.sffp ? Ld<T>::blocks(a.sffp) : 0;
  const int nb_ff = a.top * nbe + nbs;  // blocks of one sequence's feed-forward part (identity experts: skipped)
  // LDS: block table [nbv + nb_ff], vectors: v [B][nbv], feed-forward [nb_ff] of one sequence at a time
  LdBlk* tab = (LdBlk*)smem_raw;
  float* xv = (float*)(smem_raw + (size_t)(nbv + nb_ff) * sizeof(LdBlk));
  float* xf = xv + (size_t)B * nbv * BE;
  const int items = (a.W + R - 1) / R;
  for (int b = threadIdx.x; b < nbv; b += 256) {
    const int left = a.ldv / E - b * 64;
    tab[b] = LdBlk{(const T*)a.wo + (size_t)b * BE, a.ldv, left < 64 ? left : 64};
  }
  auto tile_of = [&](frag (&w)[R][U], int b0, int b1, const int (&ri)[R]) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (b0 + u < b1) {
        const LdBlk k = tab[b0 + u];
        const int c = lane < k.nch ? lane : k.nch - 1;
#pragma unroll
        for (int r = 0; r < R; ++r)
          w[r][u] = ld_nt((const frag*)((const T*)k.p + (size_t)ri[r] * k.stride) + c);
      }
    }
  };
  // first item of this wave; later items reload everything
  for (int q = 0; q < B; ++q)
    for (int i = threadIdx.x; i < nbv * BE; i += 256)
      xv[(size_t)q * nbv * BE + Ld<T>::place(i)] = i < a.n_v ? a.v[(size_t)q * a.ld_v + i] : 0.f;
  for (int it0 = blockIdx.x * 4; it0 < items; it0 += a.nwg * 4) {  // uniform per workgroup: barriers inside
    const int item = it0 + wave;
    int ri[R];
#pragma unroll
    for (int r = 0; r < R; ++r) ri[r] = item * R + r < a.W ? item * R + r : a.W - 1;
    float acc[R][B] = {};
#pragma unroll
    for (int q = 0; q < (B > 1 ? B : 1); ++q) {
      int nb = 0;  // feed-forward blocks of sequence q in the table
      if (a.moe) {
        __syncthreads();  // the part of the sequence before has been consumed
        int slot = 0;
        for (int k = 0; k < a.top; ++k) {
          const int id = a.ids[q * a.top + k];
          if (id < 0) continue;
          const float* he = a.he + (size_t)(q * a.top + k) * a.ffp;
          for (int i = threadIdx.x; i < nbe * BE; i += 256)
            xf[(size_t)slot * BE + Ld<T>::place(i)] = i < a.ffp ? he[i] : 0.f;
          for (int b = threadIdx.x; b < nbe; b += 256) {
            const int left = a.ffp / E - b * 64;
            tab[nbv + slot + b] = LdBlk{(const T*)a.down + (size_t)id * a.W * a.ffp + (size_t)b * BE, a.ffp, left < 64 ? left : 64};
          }
          slot += nbe;
        }
        if (nbs) {
          const float g = a.sh_g[q];
          for (int i = threadIdx.x; i < nbs * BE; i += 256)
            xf[(size_t)slot * BE + Ld<T>::place(i)] = i < a.sffp ? g * a.hs[(size_t)q * a.sffp + i] : 0.f;
          for (int b = threadIdx.x; b < nbs; b += 256) {
            const int left = a.sffp / E - b * 64;
            tab[nbv + slot + b] = LdBlk{(const T*)a.sdown + (size_t)b * BE, a.sffp, left < 64 ? left : 64};
          }
          slot += nbs;
        }
        nb = slot;
      }
      __syncthreads();
      const int b_lo = q == 0 ? 0 : nbv, b_hi = nbv + nb;  // the mixer part runs once, for all sequences
      frag w[R][U];
      for (int b0 = b_lo; b0 < b_hi; b0 += U) {
        tile_of(w, b0, b_hi, ri);
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int b = b0 + u;
          if (b >= b_hi) continue;
          if (b < nbv) {
#pragma unroll
            for (int j = 0; j < B; ++j) {
              const f32x4* x = (const f32x4*)(xv + ((size_t)j * nbv + b) * BE) + lane;
#pragma unroll
              for (int r = 0; r < R; ++r) acc[r][j] = ld_dot<T>(w[r][u], x, acc[r][j]);
            }
          } else {
            const f32x4* x = (const f32x4*)(xf + (size_t)(b - nbv) * BE) + lane;
#pragma unroll
            for (int r = 0; r < R; ++r) acc[r][q] = ld_dot<T>(w[r][u], x, acc[r][q]);
          }
        }
      }
    }
    ld_reduce<R, B>(acc);
    if (lane < R * B && item < items) {
      const int r = lane & (R - 1), q = lane / R, i = item * R + r;
      const float v = ld_pick<R, B>(acc, r, q);
      if (i < a.W) {
        const size_t o = (size_t)q * a.W + i;
        float y = v;
        if (a.moe) y = __builtin_fmaf(a.id_w[q], a.xn2[o], y);
        a.x_out[o] = a.x_cur[o] + y;
      }
    }
  }
}

// ---- k_ld_head ---------------------------------------------------------------------------------------------------
struct LdHeadArgs {
  const float* x;        // [B][W]
  const float *w, *b;    // final norm
  const void* head;      // [V][ld]
  float* logits;         // [B][V]
  float* part_val;       // argmax partials of sequence 0 (nullptr: none)
  int32_t* part_idx;
  int W, ld, V;
  float eps, cap;
};
template <class T, int B>
__global__ __launch_bounds__(256) void k_ld_head(const LdHeadArgs a) {
  constexpr int R = 4, U = 4;
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  float* xs = (float*)smem_raw;
  __shared__ float red[KH_WAVES_MAX];
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
  for (int q = 0; q < B; ++q) {
    float* x = xs + (size_t)q * xstride;
    float s = 0.f;
    for (int i = threadIdx.x; i < xstride; i += 256) {
      const float v = i < a.W ? a.x[(size_t)q * a.W + i] : 0.f;
      x[Ld<T>::place(i)] = v;
      s += v;
    }
    const float mean = block_sum(s, red) / (float)a.W;
    float d2 = 0.f;
    for (int i = threadIdx.x; i < a.W; i += 256) {
      const float d = x[Ld<T>::place(i)] - mean;
      d2 = __builtin_fmaf(d, d, d2);
    }
    const float rstd = 1.0f / sqrtf(block_sum(d2, red) / (float)a.W + a.eps);
    for (int i = threadIdx.x; i < a.W; i += 256)
      x[Ld<T>::place(i)] = (x[Ld<T>::place(i)] - mean) * rstd * a.w[i] + a.b[i];
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
