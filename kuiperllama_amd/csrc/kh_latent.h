// kh_latent.h — latent attention in its absorbed form.
//
// A cache row holds the normalised latent c (Rp elements, zero-padded) and the rotated key part shared by all heads
// (drp elements): q_n . (W_uk c) = (W_uk^T q_n) . c, so a query row is [W_uk^T q_n | rotated q] and every head of a
// token attends to the SAME rows; the values are the latents themselves, W_uv follows behind the softmax.  All
// H x tokens query rows of a sequence therefore share each staged key tile - one read of the cache per 16 .. 64 rows.
//
// k_latent_attn: workgroup = 4 waves = WR row tiles of 16 query rows x CP column parts (WR CP = 4) of the latent.
//   Key tiles of KT rows go straight from the cache to LDS (LDS-DMA, a ring of two).  S^T = K Q^T: a lane ends with the
//   scores of ONE query row (its column), so the running max / sum are lane scalars plus two cross-row swaps, and P^T
//   is already the second operand of O^T = C^T P^T.  The first operand, columns of the tile, comes from the same LDS
//   rows: bf16 through the transposing read (ds_read_b64_tr_b16: lane i of 16 receives element i of four rows), fp32
//   one element at a time.
// Softmax with a sink: m starts at sink_h and l at 1 in the first split (exp(sink - m), counted once, no value).
// Scores, weights and sums are fp32; P is rounded to the storage type for its product with the values.
#pragma once
#include <type_traits>

#include "kh_lgemm.h"
#include "kh_lops.h"

namespace khm {

// ---- per-token preparation: norms of the two latents, rotation of the shared key part, cache row -------------------
template <class T>
struct LatPrepArgs {
  const float* raw;        // [T][ldr]: q latent (qr), kv latent (R), rotated part (dr)
  const float *qn, *kvn;   // norm weights
  const float2* rope;      // [positions][dims / 2] (cos, sin)
  T* cq;                   // [T][ldq]
  T* cache;                // + slot * slot_elems + pos * row
  size_t slot_elems;
  int ldr, ldq, qr, R, dr, Rp, row, dims;
  float eps;
  PassTabs p;
};
template <class T>
__global__ __launch_bounds__(256) void k_latent_prep(const LatPrepArgs<T> a) {
  __shared__ float red[KH_WAVES_MAX];
  const int t = blockIdx.x;
  const float* r = a.raw + (size_t)t * a.ldr;
  const int pos = a.p.pos[t], slot = a.p.seg_slot[a.p.seg[t]];
  float s = 0.f;
  for (int i = threadIdx.x; i < a.qr; i += 256) s = __builtin_fmaf(r[i], r[i], s);
  const float rq = 1.0f / sqrtf(block_sum(s, red) / (float)a.qr + a.eps);
  for (int i = threadIdx.x; i < a.qr; i += 256) a.cq[(size_t)t * a.ldq + i] = (T)(r[i] * rq * a.qn[i]);
  r += a.qr;
  s = 0.f;
  for (int i = threadIdx.x; i < a.R; i += 256) s = __builtin_fmaf(r[i], r[i], s);
  const float rk = 1.0f / sqrtf(block_sum(s, red) / (float)a.R + a.eps);
  T* row = a.cache + (size_t)slot * a.slot_elems + (size_t)pos * a.row;
  for (int i = threadIdx.x; i < a.row; i += 256) {
    float v = 0.f;
    if (i < a.R) {
      v = r[i] * rk * a.kvn[i];
    } else if (i >= a.Rp && i - a.Rp < a.dr) {
      const int j = i - a.Rp;
      v = r[a.R + j];
      if (j < a.dims) {
        const float2 cs = a.rope[(size_t)pos * (a.dims >> 1) + (j >> 1)];
        const float o = r[a.R + (j ^ 1)];
        v = (j & 1) ? v * cs.x + o * cs.y : v * cs.x - o * cs.y;
      }
    }
    row[i] = (T)v;
  }
}

// rotated part of every head: q [T][H][dnp + drp] -> Q [T][H][Rp + drp] (pad columns zero).  grid T
template <class T>
struct RopeQArgs {
  const T* q;
  T* Q;
  const float2* rope;
  int H, dnp, dr, drp, Rp, dims;
  PassTabs p;
};
template <class T>
__global__ __launch_bounds__(256) void k_rope_q(const RopeQArgs<T> a) {
  const int t = blockIdx.x, pos = a.p.pos[t];
  for (int i = threadIdx.x; i < a.H * a.drp; i += 256) {
    const int h = i / a.drp, j = i - h * a.drp;
    const T* q = a.q + ((size_t)t * a.H + h) * (a.dnp + a.drp) + a.dnp;
    float v = j < a.dr ? (float)q[j] : 0.f;
    if (j < a.dims) {
      const float2 cs = a.rope[(size_t)pos * (a.dims >> 1) + (j >> 1)];
      const float o = (float)q[j ^ 1];
      v = (j & 1) ? v * cs.x + o * cs.y : v * cs.x - o * cs.y;
    }
    a.Q[((size_t)t * a.H + h) * (a.Rp + a.drp) + a.Rp + j] = (T)v;
  }
}

// ---- attention -------------------------------------------------------------------------------------------------
struct LatTile {  // 16 WR query rows of one segment: flattened (token, head) rows r0 ..
  int seg, r0;
};
struct LatArgs {
  const void* Q;         // [T][H][row]
  const void* cache;     // + slot * slot_elems + pos * row
  size_t slot_elems;
  const float* sink;     // [H]
  void* out;             // T [T][H][Rp] (one split)
  float* part;           // splits > 1: [T * H][splits][Rp + 4]: o (unnormalised), m, l.  One token per segment then:
                         // every row of a workgroup sees the same keys
  const LatTile* tiles;  // nullptr: one token per segment, ceil(H / rows of a tile) workgroups each
  int H, Rp, row, nsplit;
  float scale2;          // scale * log2(e)
  PassTabs p;
};

template <class T>
struct LatCfg {
  static constexpr int KT = 4 * Tile<T>::N;  // keys per tile: 32 bf16, 16 fp32 (one k-block of the second product)
};
// keys per split and splits that have any: a split gets at least KH_LAT_SPLIT_MIN keys, whole tiles
#ifndef KH_LAT_SPLIT_MIN
#define KH_LAT_SPLIT_MIN 32
#endif
__host__ __device__ __forceinline__ int lat_split_len(int n_keys, int nsplit) {
  const int per = (n_keys + nsplit - 1) / nsplit;
  return (per + KH_LAT_SPLIT_MIN - 1) / KH_LAT_SPLIT_MIN * KH_LAT_SPLIT_MIN;
}
__host__ __device__ __forceinline__ int lat_active_splits(int n_keys, int nsplit) {
  const int per = lat_split_len(n_keys, nsplit);
  return (n_keys + per - 1) / per;
}
template <class T>
static inline size_t lat_lds(int row) { return (size_t)2 * LatCfg<T>::KT * row * sizeof(T); }

// First operand of the second product: the lane's column `col`, keys 4 fh .. + 3 (and + 16 for bf16) of a tile whose
// 16-byte chunk c of row k lies in slot c ^ (k & 7)
template <int CB /* chunks per row */>
__device__ __forceinline__ bf16x8 lat_col(const char* tile, int c0, int lane, bf16) {
  typedef short s16x4 __attribute__((ext_vector_type(4)));
  const int fh = lane >> 4, k = 4 * fh + ((lane >> 2) & 3), c = (c0 >> 3) + ((lane & 3) >> 1);
  bf16x8 r;
#pragma unroll
  for (int n = 0; n < 2; ++n) {
    const int kk = k + 16 * n;
    const char* p = tile + ((size_t)kk * CB + (c ^ (kk & 7))) * 16 + (lane & 1) * 8;
    const s16x4 v = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)p);
    const bf16x4 q = __builtin_bit_cast(bf16x4, v);
#pragma unroll
    for (int i = 0; i < 4; ++i) r[4 * n + i] = q[i];
  }
  return r;
}
template <int CB>
__device__ __forceinline__ f32x4 lat_col(const char* tile, int c0, int lane, float) {
  const int fh = lane >> 4, col = c0 + (lane & 15), c = col >> 2;
  f32x4 r;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int k = 4 * fh + i;
    r[i] = *(const float*)(tile + ((size_t)k * CB + (c ^ (k & 7))) * 16 + (col & 3) * 4);
  }
  return r;
}

// RT: 16-column tiles of the latent (Rp = 16 RT); DR: rotated part / 64; CP: column parts.  The row geometry is a
// compile-time constant: a size guard around each fragment would end a scheduling block after every LDS read.
template <class T, int RT, int DR, int CP>
__global__ __launch_bounds__(256) void k_latent_attn(const LatArgs a) {
  typedef Tile<T> TL;
  typedef typename TL::frag frag;
  constexpr int E = TL::N, KT = LatCfg<T>::KT;
  constexpr int Rp = RT * 16, ROW = Rp + 64 * DR;
  constexpr int NQ = ROW / (4 * E);                            // 64-byte k-blocks of a query row
  constexpr int NT = RT / CP;                                  // latent tiles per wave
  constexpr int NS = KT / 16;                                  // score tiles
  constexpr int cblk = ROW / E, NL = KT * cblk / 256;          // chunks of a row; LDS-DMA requests per wave and tile
  constexpr int TB = KT * ROW * (int)sizeof(T);                // bytes of a tile
  extern __shared__ __attribute__((aligned(1024))) char smem_raw[];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int fr = lane & 15, fh = lane >> 4;
  const int wr = wave % (4 / CP), wc = wave / (4 / CP);
  LatTile tl;
  int n_rows, pos0, row0;
  if (a.tiles) {
    tl = a.tiles[blockIdx.x];
    n_rows = a.p.seg_n[tl.seg] * a.H;
    row0 = a.p.seg_row0[tl.seg];
  } else {  // one token per segment: no tables to wait for
    const int per = (a.H + 64 / CP - 1) / (64 / CP);
    tl.seg = (int)blockIdx.x / per;
    tl.r0 = ((int)blockIdx.x - tl.seg * per) * (64 / CP);
    n_rows = a.H;
    row0 = tl.seg;
  }
  pos0 = a.p.seg_pos0[tl.seg];
  const T* cache = (const T*)a.cache + (size_t)a.p.seg_slot[tl.seg] * a.slot_elems;
  // this lane's query row
  int r = tl.r0 + wr * 16 + fr;
  const bool live = r < n_rows;
  if (!live) r = n_rows - 1;
  const int tok = r / a.H, head = r - tok * a.H;
  const int my_pos = pos0 + tok;
  // keys [k_lo, k_hi) of this split; k_hi = 1 + the last position any row of the workgroup sees
  int rl = tl.r0 + 16 * (4 / CP) - 1;
  if (rl >= n_rows) rl = n_rows - 1;
  const int n_keys = pos0 + rl / a.H + 1;
  int k_lo = 0, k_hi = n_keys;
  if (a.nsplit > 1) {
    const int per = lat_split_len(n_keys, a.nsplit);
    k_lo = (int)blockIdx.y * per;
    if (k_lo >= n_keys) return;  // uniform; the merge does not read this split
    k_hi = k_lo + per < n_keys ? k_lo + per : n_keys;
  }
  f32x4 o[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n) o[n] = f32x4{0.f, 0.f, 0.f, 0.f};
  // ---- staging: request j of a wave covers chunks (4 j + wave) 64 .. of the tile
  int kr[NL];
  unsigned kc[NL];
#pragma unroll
  for (int j = 0; j < NL; ++j) {
    const int c = (4 * j + wave) * 64 + lane;
    kr[j] = c / cblk;
    kc[j] = (unsigned)(((c - kr[j] * cblk) ^ (kr[j] & 7)) << 4);
  }
  const unsigned lds0 = (unsigned)__builtin_amdgcn_readfirstlane((int)kh_lds_addr(smem_raw)) + 1024u * wave;
  auto issue = [&](int slot, int k0) __attribute__((always_inline)) {
    const char* base = (const char*)(cache + (size_t)k0 * ROW);
#pragma unroll
    for (int j = 0; j < NL; ++j) {
      const int k = k0 + kr[j] < n_keys ? kr[j] : n_keys - 1 - k0;  // rows behind the sequence's last may not be backed
      dma_x4_keep(base, (unsigned)(k * (ROW * (int)sizeof(T))) + kc[j], lds0 + (unsigned)(slot * TB + 4096 * j));
    }
  };
  if (k_lo < k_hi) issue(0, k_lo);
  const char* qrow = (const char*)((const T*)a.Q + ((size_t)(row0 + tok) * a.H + head) * ROW) + 16 * fh;
  frag fq[NQ];
#pragma unroll
  for (int b = 0; b < NQ; ++b) fq[b] = *(const frag*)(qrow + 64 * b);
  const bool sinks = (a.nsplit == 1 || blockIdx.y == 0);
  float m = sinks ? a.sink[head] * 1.44269504088896f : -INFINITY, l = sinks && fh == 0 ? 1.f : 0.f;
  int slot = 0;
  for (int k0 = k_lo; k0 < k_hi; k0 += KT, slot ^= 1) {
    wait_vm<0>();     // this tile has landed (the next one is requested behind the barrier)
    __syncthreads();  // ... for every wave, and everyone is done with the tile before
    if (k0 + KT < k_hi) issue(slot ^ 1, k0 + KT);
    const char* Kt = smem_raw + slot * TB;
    f32x4 s[NS];
#pragma unroll
    for (int n = 0; n < NS; ++n) s[n] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int b = 0; b < NQ; ++b)
#pragma unroll
      for (int n = 0; n < NS; ++n) {
        const int k = n * 16 + fr;
        const frag fk = *(const frag*)(Kt + ((size_t)k * cblk + ((4 * b + fh) ^ (k & 7))) * 16);
        s[n] = TL::mma(fk, fq[b], s[n]);
      }
    // lane: keys k0 + 16 n + 4 fh + i of row r
    float mx = m;
#pragma unroll
    for (int n = 0; n < NS; ++n)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int k = k0 + 16 * n + 4 * fh + i;
        s[n][i] = k <= my_pos && k < k_hi ? s[n][i] * a.scale2 : -INFINITY;
        mx = fmaxf(mx, s[n][i]);
      }
    mx = xor16_max(mx);
    mx = xor32_max(mx);
    const float base = mx == -INFINITY ? 0.f : mx;  // nothing seen yet by this row
    const float f = __builtin_amdgcn_exp2f(m - base);
    m = mx;
    l *= f;
    frag p;
#pragma unroll
    for (int n = 0; n < NS; ++n)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float e = __builtin_amdgcn_exp2f(s[n][i] - base);
        l += e;
        p[4 * n + i] = (T)e;
      }
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const frag fv = lat_col<cblk>(Kt, (wc * NT + n) * 16, lane, T());
#pragma unroll
      for (int i = 0; i < 4; ++i) o[n][i] *= f;
      o[n] = TL::mma(fv, p, o[n]);
    }
  }
  l = xor16_sum(l);
  l = xor32_sum(l);
  if (!live) return;
  const size_t orow = (size_t)(row0 + tok) * a.H + head;
  if (a.nsplit == 1) {
    const float inv = 1.0f / l;
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const int c0 = (wc * NT + n) * 16;
      f32x4 v;
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = o[n][i] * inv;
      *(typename TL::quad*)((T*)a.out + orow * Rp + c0 + 4 * fh) = to_quad<T>(v);
    }
  } else {
    float* p = a.part + (orow * a.nsplit + blockIdx.y) * (size_t)(Rp + 4);
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const int c0 = (wc * NT + n) * 16;
      *(f32x4*)(p + c0 + 4 * fh) = o[n];
    }
    if (wc == 0 && fh == 0) {
      p[Rp] = m;
      p[Rp + 1] = l;
    }
  }
}

template <class T>
int lat_attn_launch(hipStream_t s, const LatArgs& a, int ntiles, int cp) {
  const size_t lds = lat_lds<T>(a.row);
  auto go = [&](auto kern) -> int {
    if (lds > 64 * 1024) {
      const hipError_t e = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      if (e != hipSuccess) return (int)e;
    }
    hipLaunchKernelGGL(kern, dim3(ntiles, a.nsplit), dim3(256), lds, s, a);
    return KH_OK;
  };
  // column parts: 4 = 16-row tiles, 2 = 32-row tiles (latents of more than 256), 1 = 64-row tiles
  auto pick = [&](auto dr) -> int {
    constexpr int DR = decltype(dr)::value;
    if (cp == 4) {
      if (a.Rp == 64) return go(k_latent_attn<T, 4, DR, 4>);
      if (a.Rp == 128) return go(k_latent_attn<T, 8, DR, 4>);
      if (a.Rp == 256) return go(k_latent_attn<T, 16, DR, 4>);
      if (a.Rp == 512) return go(k_latent_attn<T, 32, DR, 4>);
    } else if (cp == 2) {
      if (a.Rp == 512) return go(k_latent_attn<T, 32, DR, 2>);
    } else if (cp == 1) {
      if (a.Rp == 64) return go(k_latent_attn<T, 4, DR, 1>);
      if (a.Rp == 128) return go(k_latent_attn<T, 8, DR, 1>);
      if (a.Rp == 256) return go(k_latent_attn<T, 16, DR, 1>);
    }
    return KH_ERR_UNSUPPORTED;
  };
  if (a.row - a.Rp == 64) return pick(std::integral_constant<int, 1>());
  if (a.row - a.Rp == 128) return pick(std::integral_constant<int, 2>());
  return KH_ERR_UNSUPPORTED;
}
// padded sizes of a cache row the kernel is instantiated for: latent and rotated part (0: none)
static inline int lat_pad_latent(int R) { return R <= 64 ? 64 : (R <= 128 ? 128 : (R <= 256 ? 256 : (R <= 512 ? 512 : 0))); }
static inline int lat_pad_rot(int dr) { return dr <= 64 ? 64 : (dr <= 128 ? 128 : 0); }
}  // namespace khm
