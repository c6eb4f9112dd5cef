// kh_heads.h — attention over cached keys and values with grouped heads (query head h reads key / value head h / (H / G)):
// per-head RMS norms of queries and keys, a learned bias by distance, sliding windows, chunks, a sink, an output gate.
// Everything but the kernel's tile sizes is a parameter.
//
// A cache row holds, key / value head by head, [key (dkp) | value (dvp)], both padded to 64 elements with zeros.  A run
// keeps `ring` rows per sequence: position p lies in row p % ring (ring = the cache length where every key stays
// visible; for windows and chunks the span of one query plus the tokens of one pass).
//
// k_heads_attn: workgroup = 4 waves = WR x MR tiles of 16 query rows x CP column parts (WR CP = 4) of the values of ONE
//   key / value head; a query row is a (token, query head of the group) pair, so the group's heads share each staged key
//   tile.  Tiles of KT cache rows go straight to LDS (LDS-DMA, a ring of NST stages).  S^T = K Q^T: a lane ends with the scores
//   of ONE query row per tile of 16, so the running max / sum are lane scalars plus two cross-row swaps, and P^T is
//   already the second operand of O^T = V^T P^T, whose first operand comes from the same LDS rows (lat_col).
//   Queries are read as projected and normalised in registers; scale and log2(e) are folded in with the norm weights.
// Scores, weights and sums are fp32; queries and P are rounded to the storage type for their products.
#pragma once
#include "kh_latent.h"

namespace khm {

// Keys position `pos` sees: [first(pos), pos].  0: no limit of that kind.
struct KeySpan {
  int window;  // at most that many keys, itself included
  int chunk;   // only keys of its own chunk, counted from position 0 of the sequence
  __host__ __device__ __forceinline__ int first(int pos) const {
    int f = chunk > 0 ? pos - pos % chunk : 0;
    if (window > 0 && pos - window + 1 > f) f = pos - window + 1;
    return f;
  }
};

// ---- cache rows: one wave per (token, key / value head) ----------------------------------------------------------------
struct HeadRow {
  const float* kn;  // [dkp] norm weight behind the keys' RMS norm (nullptr: no norm)
  int G, dk, dv, dkr, dvr, dkp, dvp, k_off, v_off, ring;  // k_off, v_off: first key / value column of a projected row
  float eps;
};
template <class R, class T>
__device__ __forceinline__ void heads_cache_row(const HeadRow& a, const R* raw, T* cache, int pos, int g, int lane) {
  constexpr int N = 4;  // 64 N >= the largest padded head
  const R *k = raw + a.k_off + (size_t)g * a.dkr, *v = raw + a.v_off + (size_t)g * a.dvr;
  float x[N], w[N], y[N], s = 0.f;
#pragma unroll
  for (int j = 0; j < N; ++j) {
    const int i = 64 * j + lane;
    x[j] = i < a.dk ? (float)k[i] : 0.f;
    y[j] = i < a.dv ? (float)v[i] : 0.f;
    w[j] = a.kn && i < a.dkp ? a.kn[i] : 1.f;
    s = __builtin_fmaf(x[j], x[j], s);
  }
  const float rs = a.kn ? 1.0f / sqrtf(wave_sum(s) / (float)a.dk + a.eps) : 1.f;
  T* row = cache + ((size_t)(pos % a.ring) * a.G + g) * (a.dkp + a.dvp);
#pragma unroll
  for (int j = 0; j < N; ++j) {
    const int i = 64 * j + lane;
    if (i < a.dkp) row[i] = (T)(x[j] * rs * w[j]);
    if (i < a.dvp) row[a.dkp + i] = (T)y[j];
  }
}
template <class T>
struct HeadRowsArgs {
  HeadRow r;
  const T* raw;  // [tokens][ldr]
  T* cache;      // + slot * slot_elems
  size_t slot_elems;
  int ldr, T_all;
  PassTabs p;
};
// grid (tokens G / 4)
template <class T>
__global__ __launch_bounds__(256) void k_heads_rows(const HeadRowsArgs<T> a) {
  const int i = blockIdx.x * 4 + (threadIdx.x >> 6), t = i / a.r.G, g = i - t * a.r.G;
  if (t >= a.T_all) return;
  heads_cache_row(a.r, a.raw + (size_t)t * a.ldr, a.cache + (size_t)a.p.seg_slot[a.p.seg[t]] * a.slot_elems, a.p.pos[t], g,
                  threadIdx.x & 63);
}

// ---- attention -------------------------------------------------------------------------------------------------
struct HeadsArgs {
  const void* raw;       // [T][ldr] projected rows: query heads dkr apart from column 0; gate logits dvr apart from g_off
  int raw_f32;           // the rows are fp32 (else the storage type)
  int g_off;             // -1: no output gate (it is applied where the result is written: with one split)
  const float* qn;       // [dkp] query norm weight (nullptr: no norm)
  const void* cache;     // + slot * slot_elems + row * G (dkp + dvp)
  size_t slot_elems;
  const float* bias;     // [H][nbias] by distance, in units of log2(e); the last entry holds for everything beyond.  nullptr: none
  void* out;             // T [T][ldo], heads dvr apart (one split)
  float* part;           // splits > 1: [T H][splits][dvp + 4]: o (unnormalised), m, l.  One token per segment then
  const LatTile* tiles;  // nullptr: one token per segment, ceil((H / G) / rows of a tile) workgroups each
  int H, G, dk, dkr, dkp, dvr, dvp, ldr, ldo, ring, nsplit, nbias, bias_lds;
  int sink;              // the softmax denominator has one more term exp(0) without a value
  KeySpan span;
  float eps, scale2;     // scale * log2(e)
  PassTabs p;
};

// KN, KV: key and value size in units of 64.  CP = 4: 16 rows per workgroup; CP = 1: 64 MR rows.
// Two waves per SIMD where the accumulators allow it: within 256 registers the compiler keeps them where the rescaling can
// reach them (beyond, it moves them between two register files in every tile).
template <class T, int KN, int KV, int CP, int MR>
__global__ __launch_bounds__(256, KN + KV > 4 ? 1 : 2) void k_heads_attn(const HeadsArgs a) {
  typedef Tile<T> TL;
  typedef typename TL::frag frag;
  constexpr int E = TL::N, KT = 4 * E, NS = KT / 16, ES = (int)sizeof(T);
  constexpr int DK = 64 * KN, DV = 64 * KV, ROW = DK + DV, CB = ROW / E;
  constexpr int NQ = DK / (4 * E), NT = DV / 16 / CP, NL = ROW / 64;
  constexpr int TB = KT * ROW * ES, NST = TB <= 24 * 1024 ? 3 : 2, WR = 4 / CP, ROWS = 16 * MR * WR;
  extern __shared__ __attribute__((aligned(1024))) char smem_raw[];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int fr = lane & 15, fh = lane >> 4, wr = wave % WR, wc = wave / WR;
  const int g = blockIdx.x, per = a.H / a.G;
  LatTile tl;
  int n_rows, row0;
  if (a.tiles) {
    // longest key ranges first; a launch of at most two workgroups per CU pairs the longest with the shortest instead
    const int nt = (int)gridDim.y, half = (nt + 1) >> 1, y = (int)blockIdx.y;
    tl = a.tiles[nt * a.G <= 512 && y >= half ? nt - 1 - (y - half) : y];
    n_rows = a.p.seg_n[tl.seg] * per;
    row0 = a.p.seg_row0[tl.seg];
  } else {
    const int nt = (per + ROWS - 1) / ROWS;
    tl.seg = (int)blockIdx.y / nt;
    tl.r0 = ((int)blockIdx.y - tl.seg * nt) * ROWS;
    n_rows = per;
    row0 = tl.seg;
  }
  const int pos0 = a.p.seg_pos0[tl.seg];
  const char* cache = (const char*)((const T*)a.cache + (size_t)a.p.seg_slot[tl.seg] * a.slot_elems + (size_t)g * ROW);
  // the lane's query rows
  int head[MR], tok[MR], my_pos[MR];
  bool live[MR];
#pragma unroll
  for (int q = 0; q < MR; ++q) {
    int r = tl.r0 + (wr * MR + q) * 16 + fr;
    live[q] = r < n_rows;
    if (!live[q]) r = n_rows - 1;
    tok[q] = r / per;
    head[q] = g * per + r - tok[q] * per;
    my_pos[q] = pos0 + tok[q];
  }
  auto pos_of = [&](int r) __attribute__((always_inline)) { return pos0 + (r < n_rows ? r : n_rows - 1) / per; };
  // positions of the first and last row of the wave; keys [k_lo, k_hi) of the workgroup
  const int p_lo = pos_of(tl.r0 + wr * MR * 16), p_hi = pos_of(tl.r0 + (wr + 1) * MR * 16 - 1);
  const int w_first = a.span.first(p_lo), w_full = a.span.first(p_hi);  // some row sees from, every row sees from
  const int n_keys = pos_of(tl.r0 + ROWS - 1) + 1;
  int k_lo = a.span.first(pos_of(tl.r0)), k_hi = n_keys;
  if (a.nsplit > 1) {
    const int len = lat_split_len(n_keys - k_lo, a.nsplit);
    k_lo += (int)blockIdx.z * len;
    if (k_lo >= n_keys) return;  // uniform; the merge does not read this split
    k_hi = k_lo + len < n_keys ? k_lo + len : n_keys;
  }
  int my_first[MR];
#pragma unroll
  for (int q = 0; q < MR; ++q) my_first[q] = a.span.first(my_pos[q]);
  // ---- queries: norm and scale in registers (a row's elements lie in the four lanes fr, fr + 16, ...)
  frag fq[MR][NQ];
#pragma unroll
  for (int q = 0; q < MR; ++q) {
    float x[NQ][E], s = 0.f;
    const size_t at = (size_t)(row0 + tok[q]) * a.ldr + (size_t)head[q] * a.dkr;
#pragma unroll
    for (int b = 0; b < NQ; ++b) {
      const int e0 = 4 * E * b + E * fh;  // dkr is a multiple of 16: a fragment is inside or outside as a whole
      if (a.raw_f32) {
#pragma unroll
        for (int i = 0; i < E; i += 4) {
          const f32x4 v = e0 < a.dkr ? *(const f32x4*)((const float*)a.raw + at + e0 + i) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int j = 0; j < 4; ++j) x[b][i + j] = v[j];
        }
      } else {
        const bool in = e0 < a.dkr;
        const frag v = *(const frag*)((const T*)a.raw + at + (in ? e0 : 0));
#pragma unroll
        for (int i = 0; i < E; ++i) x[b][i] = in ? (float)v[i] : 0.f;
      }
#pragma unroll
      for (int i = 0; i < E; ++i) s = __builtin_fmaf(x[b][i], x[b][i], s);
    }
    s = xor16_sum(s);
    s = xor32_sum(s);
    const float f = a.qn ? a.scale2 / sqrtf(s / (float)a.dk + a.eps) : a.scale2;
#pragma unroll
    for (int b = 0; b < NQ; ++b)
#pragma unroll
      for (int i = 0; i < E; i += 4) {
        const f32x4 w = a.qn ? *(const f32x4*)(a.qn + 4 * E * b + E * fh + i) : f32x4{1.f, 1.f, 1.f, 1.f};
#pragma unroll
        for (int j = 0; j < 4; ++j) fq[q][b][i + j] = (T)(x[b][i + j] * f * w[j]);
      }
  }
  // ---- distance bias: the group's rows of the table to LDS when a key of this workgroup is near enough to need them
  float* tab = (float*)(smem_raw + NST * TB);
  float far[MR];
#pragma unroll
  for (int q = 0; q < MR; ++q) far[q] = a.bias ? a.bias[(size_t)head[q] * a.nbias + a.nbias - 1] : 0.f;
  if (a.bias && a.bias_lds && pos_of(tl.r0) - (k_hi - 1) < a.nbias - 1)
    for (int i = threadIdx.x; i < per * a.nbias; i += 256) tab[i] = a.bias[(size_t)g * per * a.nbias + i];
  // ---- staging: request j of a wave covers chunks (4 j + wave) 64 .. of the tile; slot s of row r holds chunk s ^ (r & 7)
  int kr[NL];
  unsigned kc[NL];
#pragma unroll
  for (int j = 0; j < NL; ++j) {
    const int c = (4 * j + wave) * 64 + lane;
    kr[j] = c / CB;
    kc[j] = (unsigned)(((c - kr[j] * CB) ^ (kr[j] & 7)) << 4);
  }
  const unsigned lds0 = (unsigned)__builtin_amdgcn_readfirstlane((int)kh_lds_addr(smem_raw)) + 1024u * wave;
  const unsigned row_b = (unsigned)(a.G * ROW * ES);
  int fill_row = k_lo % a.ring;  // cache row of the next tile to request
  auto issue = [&](int slot, int k0) __attribute__((always_inline)) {
#pragma unroll
    for (int j = 0; j < NL; ++j) {
      const int k = k0 + kr[j] < n_keys ? kr[j] : n_keys - 1 - k0;  // rows behind the sequence's last may not be backed
      int r = fill_row + k;
      r = r < a.ring ? r : r - a.ring;
      dma_x4_keep(cache, (unsigned)r * row_b + kc[j], lds0 + (unsigned)(slot * TB + 4096 * j));
    }
    fill_row += KT;
    if (fill_row >= a.ring) fill_row -= a.ring;
  };
  float m[MR], l[MR];
  f32x4 o[MR][NT];
#pragma unroll
  for (int q = 0; q < MR; ++q) {
    const bool sinks = a.sink && (a.nsplit == 1 || blockIdx.z == 0);
    m[q] = sinks ? 0.f : -1e30f;  // finite: a row without a visible key yet keeps weights of zero, not NaN
    l[q] = sinks && fh == 0 ? 1.f : 0.f;
#pragma unroll
    for (int n = 0; n < NT; ++n) o[q][n] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
#pragma unroll
  for (int i = 0; i < NST - 1; ++i)
    if (k_lo + i * KT < k_hi) issue(i, k_lo + i * KT);
  int slot = -1, fill = NST - 2;
  for (int k0 = k_lo; k0 < k_hi; k0 += KT) {
    slot = slot + 1 == NST ? 0 : slot + 1;
    fill = fill + 1 == NST ? 0 : fill + 1;
    // this stage has landed when only the younger NST - 2 stages are outstanding
    if (k0 + (NST - 2) * KT < k_hi) wait_vm<(NST - 2) * NL>();
    else wait_vm<0>();
    __syncthreads();
    if (k0 + (NST - 1) * KT < k_hi) issue(fill, k0 + (NST - 1) * KT);
    if (k0 > p_hi || k0 + KT <= w_first) continue;  // nothing in this tile for the wave (barriers stay uniform)
    const char* Kt = smem_raw + slot * TB;
    f32x4 s[MR][NS];
#pragma unroll
    for (int q = 0; q < MR; ++q)
#pragma unroll
      for (int n = 0; n < NS; ++n) s[q][n] = f32x4{0.f, 0.f, 0.f, 0.f};
    frag fk[NQ][NS];
#pragma unroll
    for (int b = 0; b < NQ; ++b)
#pragma unroll
      for (int n = 0; n < NS; ++n) {
        const int k = n * 16 + fr;
        fk[b][n] = *(const frag*)(Kt + ((size_t)k * CB + ((4 * b + fh) ^ (k & 7))) * 16);
      }
    frag fv[NT];  // requested with the keys: they arrive under the scores and the softmax
#pragma unroll
    for (int n = 0; n < NT; ++n) fv[n] = lat_col<CB>(Kt, DK + (wc * NT + n) * 16, lane, T());
#pragma unroll
    for (int b = 0; b < NQ; ++b)
#pragma unroll
      for (int n = 0; n < NS; ++n)
#pragma unroll
        for (int q = 0; q < MR; ++q) s[q][n] = TL::mma(fk[b][n], fq[q][b], s[q][n]);
    // lane: keys k0 + 16 n + 4 fh + i of its rows
    frag p[MR];
    const bool edge = k0 + KT - 1 > p_lo || k0 < w_full || k0 + KT > k_hi;
    const bool near = a.bias && p_lo - (k0 + KT - 1) < a.nbias - 1;
#pragma unroll
    for (int q = 0; q < MR; ++q) {
      if (near) {  // two loads of known address space, not one of a selected address
        const int d0 = my_pos[q] - k0 - 4 * fh;
        auto add = [&](const float* row) __attribute__((always_inline)) {
#pragma unroll
          for (int n = 0; n < NS; ++n)
#pragma unroll
            for (int i = 0; i < 4; ++i) s[q][n][i] += row[min(max(d0 - 16 * n - i, 0), a.nbias - 1)];
        };
        if (a.bias_lds) add(tab + (head[q] - g * per) * a.nbias);
        else add(a.bias + (size_t)head[q] * a.nbias);
      }
      if (edge) {
#pragma unroll
        for (int n = 0; n < NS; ++n)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int k = k0 + 16 * n + 4 * fh + i;
            s[q][n][i] = k <= my_pos[q] && k >= my_first[q] && k < k_hi ? s[q][n][i] : -INFINITY;
          }
      }
      const float add = near ? 0.f : far[q];  // the same for every key of a far tile: joins the maximum
      float mx = s[q][0][0];
#pragma unroll
      for (int n = 0; n < NS; ++n)
#pragma unroll
        for (int i = 0; i < 4; ++i) mx = fmaxf(mx, s[q][n][i]);
      mx += add;
      // the running maximum rarely moves after the first tiles: rescale only when some row's does
      if (__any(mx > m[q])) {
        mx = fmaxf(mx, m[q]);
        mx = xor16_max(mx);
        mx = xor32_max(mx);
        const float f = __builtin_amdgcn_exp2f(m[q] - mx);
        m[q] = mx;
        l[q] *= f;
#pragma unroll
        for (int n = 0; n < NT; ++n)
#pragma unroll
          for (int i = 0; i < 4; ++i) o[q][n][i] *= f;
      }
      const float base = m[q] - add;
      float sum = 0.f;
#pragma unroll
      for (int n = 0; n < NS; ++n)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float e = __builtin_amdgcn_exp2f(s[q][n][i] - base);
          sum += e;
          p[q][4 * n + i] = (T)e;
        }
      l[q] += sum;
    }
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
      for (int q = 0; q < MR; ++q) o[q][n] = TL::mma(fv[n], p[q], o[q][n]);
  }
#pragma unroll
  for (int q = 0; q < MR; ++q) {
    float sum = xor16_sum(l[q]);
    sum = xor32_sum(sum);
    if (!live[q]) continue;
    if (a.nsplit == 1) {
      const float inv = 1.0f / sum;
      const size_t t = (size_t)(row0 + tok[q]);
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        const int c = (wc * NT + n) * 16 + 4 * fh;
        if (c >= a.dvr) continue;
        f32x4 v;
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = o[q][n][i] * inv;
        if (a.g_off >= 0) {
          const size_t at = t * a.ldr + a.g_off + (size_t)head[q] * a.dvr + c;
          const f32x4 z = a.raw_f32 ? *(const f32x4*)((const float*)a.raw + at) : quad_f((const T*)a.raw + at);
#pragma unroll
          for (int i = 0; i < 4; ++i) v[i] *= sigmoid1(z[i]);
        }
        *(typename TL::quad*)((T*)a.out + t * a.ldo + (size_t)head[q] * a.dvr + c) = to_quad<T>(v);
      }
    } else {
      float* pt = a.part + (((size_t)(row0 + tok[q]) * a.H + head[q]) * a.nsplit + blockIdx.z) * (size_t)(DV + 4);
#pragma unroll
      for (int n = 0; n < NT; ++n) *(f32x4*)(pt + (wc * NT + n) * 16 + 4 * fh) = o[q][n];
      if (wc == 0 && fh == 0) {
        pt[DV] = m[q];
        pt[DV + 1] = sum;
      }
    }
  }
}

#define KH_HEADS_MAX_DIM 256
#define KH_HEADS_BIAS_LDS (32 * 1024)
// rows of a workgroup's tile: 16, 64 or, for bf16 heads of up to 128, 128 (two row tiles per wave share every operand)
static inline bool heads_wide_rows(int dkp, int dvp, size_t elem) { return elem == 2 && dkp <= 128 && dvp <= 128; }
template <class T>
int heads_attn_launch(hipStream_t s, HeadsArgs a, int ntiles, int rows);
extern template int heads_attn_launch<bf16>(hipStream_t, HeadsArgs, int, int);
extern template int heads_attn_launch<float>(hipStream_t, HeadsArgs, int, int);
}  // namespace khm
