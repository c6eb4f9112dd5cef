// kh_expanded.h — latent attention of long prompt segments in its expanded form.
//
// The absorbed form (kh_latent.h) contracts kv_rank + rot_dim per score; a prompt segment instead rebuilds its heads'
// keys W_uk c and values W_uv c once per pass (two GEMMs over the cached latents) and contracts dim + rot_dim.  The
// values are produced TRANSPOSED ([head value column][key]: the GEMM with its operands swapped), so every operand of
// the attention kernel is a row of consecutive bytes and all staging is LDS-DMA.
//
// k_expanded_attn: workgroup = 4 waves x MR tiles of 16 tokens of ONE head; key tiles of KT (a 64-byte row of the
// transposed values) through a ring of KH_EXP_STAGES LDS stages.  S^T = K Q^T and O^T = V^T P^T as in kh_latent.h; here the key order is
// permuted where the K fragments are read (score tile n, row 4 h + i <- key 8 h + 4 n + i for bf16).
#pragma once
#include "kh_latent.h"
#include "kh_lgemm.h"

#ifndef KH_EXP_STAGES
#define KH_EXP_STAGES 3
#endif

namespace khm {

struct ExpArgs {
  const void* Q;       // [T][H][dnp + drp], rotated
  const void* Kx;      // [keys][H dnp]
  const void* Vx;      // [H dvp][ldv]
  const void* cache;   // rotated key parts: row k at + k * row (already offset to the part's first column)
  const float* sink;
  void* out;           // T [T][H dvp]
  int H, dnp, drp, dvp, row, ldv;
  int row0, n, pos0;   // the segment's rows in Q / out, their number, position of the first
  float scale2;        // > 0
};

// KN, KR, KV: unrotated key part, rotated part and value size in units of 64 (compile-time: see kh_latent.h)
template <class T, int KN, int KR, int KV, int MR>
__global__ __launch_bounds__(256) void k_expanded_attn(const ExpArgs a) {
  typedef Tile<T> TL;
  typedef typename TL::frag frag;
  constexpr int E = TL::N, KT = 4 * E, NS = KT / 16, ES = (int)sizeof(T);
  constexpr int DN = 64 * KN, DRP = 64 * KR, DV = 64 * KV, NQ = (DN + DRP) / (4 * E), NV = DV / 16;
  extern __shared__ __attribute__((aligned(1024))) char smem_raw[];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int fr = lane & 15, fh = lane >> 4;
  const int head = blockIdx.x;
  // longest key ranges first; a launch of at most two workgroups per CU pairs the longest with the shortest instead
  const int nt = (int)gridDim.y, half = (nt + 1) >> 1, by = (int)blockIdx.y;
  const int tile = nt * (int)gridDim.x <= 512 && by >= half ? by - half : nt - 1 - by;
  const int q0 = tile * (64 * MR);
  constexpr int qc = DN / E, rc = DRP / E;  // 16-byte chunks of the key parts
  constexpr int bytes_k = KT * DN * ES, bytes_r = KT * DRP * ES, stage = bytes_k + bytes_r + DV * 64;
  int q_last = q0 + 64 * MR - 1;
  q_last = q_last < a.n ? q_last : a.n - 1;
  const int n_keys = a.pos0 + q_last + 1;
  const T* Q = (const T*)a.Q;
  frag fq[MR][NQ];
  int my_pos[MR];
#pragma unroll
  for (int m = 0; m < MR; ++m) {
    int t = q0 + (wave * MR + m) * 16 + fr;
    t = t < a.n ? t : a.n - 1;
    my_pos[m] = a.pos0 + t;
    const char* q = (const char*)(Q + ((size_t)(a.row0 + t) * a.H + head) * (DN + DRP)) + 16 * fh;
#pragma unroll
    for (int b = 0; b < NQ; ++b) fq[m][b] = *(const frag*)(q + 64 * b);
  }
  const unsigned lds0 = (unsigned)__builtin_amdgcn_readfirstlane((int)kh_lds_addr(smem_raw));
  // slot s of a row of `c` chunks (c >= 8) holds chunk s ^ swz(row)
  auto swz = [](int row) __attribute__((always_inline)) { return (row & 3) | ((row >> 1) & 4); };
  // LDS-DMA requests of a wave and stage (64 chunks each): request j covers chunks (4 j + wave) 64 ..
  constexpr int nK = KT * qc / 256, nR = KT * rc / 256, nV = DV * 4 / 256, NL = nK + nR + nV;
  unsigned vk[nK], vr[nR], vv[nV];
  int rr[nR];
#pragma unroll
  for (int j = 0; j < nK; ++j) {
    const int c = (4 * j + wave) * 64 + lane, r = c / qc, s = c - r * qc;
    vk[j] = (unsigned)(r * a.H * DN * ES + ((s ^ swz(r)) << 4));
  }
#pragma unroll
  for (int j = 0; j < nR; ++j) {
    const int c = (4 * j + wave) * 64 + lane, r = c / rc, s = c - r * rc;
    rr[j] = r;
    vr[j] = (unsigned)((s ^ swz(r)) << 4);
  }
#pragma unroll
  for (int j = 0; j < nV; ++j) {
    const int c = (4 * j + wave) * 64 + lane;
    vv[j] = (unsigned)((c >> 2) * a.ldv * ES + ((c & 3) << 4));
  }
  auto issue = [&](int slot, int k0) __attribute__((always_inline)) {
    const unsigned d0 = lds0 + (unsigned)(slot * stage) + 1024u * wave;
    const char* kb = (const char*)a.Kx + ((size_t)k0 * a.H + head) * DN * ES;
#pragma unroll
    for (int j = 0; j < nK; ++j) dma_x4_keep(kb, vk[j], d0 + 4096u * j);
#pragma unroll
    for (int j = 0; j < nR; ++j) {
      const int k = k0 + rr[j] < n_keys ? k0 + rr[j] : n_keys - 1;  // rows behind the sequence's last are not backed
      dma_x4_keep(a.cache, (unsigned)(k * a.row * ES) + vr[j], d0 + bytes_k + 4096u * j);
    }
    const char* vb = (const char*)a.Vx + ((size_t)head * DV * a.ldv + k0) * ES;
#pragma unroll
    for (int j = 0; j < nV; ++j) dma_x4_keep(vb, vv[j], d0 + bytes_k + bytes_r + 4096u * j);
  };
  float m[MR], l[MR];
  f32x4 o[MR][NV];
#pragma unroll
  for (int q = 0; q < MR; ++q) {
    m[q] = a.sink[head] * 1.44269504088896f;
    l[q] = fh == 0 ? 1.f : 0.f;
#pragma unroll
    for (int n = 0; n < NV; ++n) o[q][n] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const int wave_last = a.pos0 + q0 + (wave + 1) * MR * 16 - 1;  // last position any row of this wave sees
  constexpr int NST = KH_EXP_STAGES;
#pragma unroll
  for (int i = 0; i < NST - 1; ++i)
    if (i * KT < n_keys) issue(i, i * KT);
  int slot = -1, fill = NST - 2;
  for (int k0 = 0; k0 < n_keys; k0 += KT) {
    slot = slot + 1 == NST ? 0 : slot + 1;
    fill = fill + 1 == NST ? 0 : fill + 1;
    // this stage has landed when only the younger NST - 2 stages are outstanding
    if (k0 + (NST - 2) * KT < n_keys) wait_vm<(NST - 2) * NL>();
    else wait_vm<0>();
    __syncthreads();
    if (k0 + (NST - 1) * KT < n_keys) issue(fill, k0 + (NST - 1) * KT);
    if (k0 > wave_last) continue;  // nothing in this tile for the wave (barriers stay uniform)
    const char* Kt = smem_raw + slot * stage;
    const char* Rt = Kt + bytes_k;
    const char* Vt = Rt + bytes_r;
    // keys, then values, are requested from LDS together: the values arrive under the scores and the softmax
    frag fk[NQ][NS], fv[NV];
#pragma unroll
    for (int b = 0; b < NQ; ++b) {
      const int c = 4 * b + fh;
#pragma unroll
      for (int n = 0; n < NS; ++n) {
        const int k = NS == 2 ? 8 * (fr >> 2) + 4 * n + (fr & 3) : fr;
        fk[b][n] = *(const frag*)(4 * b < qc ? Kt + ((size_t)k * qc + (c ^ swz(k))) * 16 : Rt + ((size_t)k * rc + ((c - qc) ^ swz(k))) * 16);
      }
    }
#pragma unroll
    for (int n = 0; n < NV; ++n) fv[n] = *(const frag*)(Vt + (size_t)(n * 16 + fr) * 64 + (fh << 4));
    __builtin_amdgcn_sched_barrier(0);
    f32x4 s[MR][NS];
#pragma unroll
    for (int q = 0; q < MR; ++q)
#pragma unroll
      for (int n = 0; n < NS; ++n) s[q][n] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int b = 0; b < NQ; ++b)
#pragma unroll
      for (int n = 0; n < NS; ++n)
#pragma unroll
        for (int q = 0; q < MR; ++q) s[q][n] = TL::mma(fk[b][n], fq[q][b], s[q][n]);
    frag p[MR];
    const bool edge = k0 + KT - 1 > a.pos0 + q0 + wave * MR * 16;  // the tile crosses the diagonal of some row
#pragma unroll
    for (int q = 0; q < MR; ++q) {
      if (edge) {
#pragma unroll
        for (int n = 0; n < NS; ++n)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int k = k0 + (NS == 2 ? 8 * fh + 4 * n + i : 4 * fh + i);
            s[q][n][i] = k <= my_pos[q] ? s[q][n][i] : -INFINITY;
          }
      }
      float mx = s[q][0][0];
#pragma unroll
      for (int n = 0; n < NS; ++n)
#pragma unroll
        for (int i = 0; i < 4; ++i) mx = fmaxf(mx, s[q][n][i]);
      mx *= a.scale2;
      // the running maximum (at least the sink) rarely moves after the first tiles: rescale only when some row's does
      if (__any(mx > m[q])) {
        mx = fmaxf(mx, m[q]);
        mx = xor16_max(mx);
        mx = xor32_max(mx);
        const float f = __builtin_amdgcn_exp2f(m[q] - mx);
        m[q] = mx;
        l[q] *= f;
#pragma unroll
        for (int n = 0; n < NV; ++n)
#pragma unroll
          for (int i = 0; i < 4; ++i) o[q][n][i] *= f;
      }
      float sum = 0.f;
#pragma unroll
      for (int n = 0; n < NS; ++n)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float e = __builtin_amdgcn_exp2f(__builtin_fmaf(s[q][n][i], a.scale2, -m[q]));
          sum += e;
          p[q][4 * n + i] = (T)e;
        }
      l[q] += sum;
    }
#pragma unroll
    for (int n = 0; n < NV; ++n)
#pragma unroll
      for (int q = 0; q < MR; ++q) o[q][n] = TL::mma(fv[n], p[q], o[q][n]);
  }
#pragma unroll
  for (int q = 0; q < MR; ++q) {
    float sum = xor16_sum(l[q]);
    sum = xor32_sum(sum);
    const float inv = 1.0f / sum;
    const int t = q0 + (wave * MR + q) * 16 + fr;
    if (t >= a.n) continue;
    T* out = (T*)a.out + ((size_t)(a.row0 + t) * a.H + head) * DV + 4 * fh;
#pragma unroll
    for (int n = 0; n < NV; ++n) {
        f32x4 v;
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = o[q][n][i] * inv;
        *(typename TL::quad*)(out + n * 16) = to_quad<T>(v);
    }
  }
}

// in-place rotation of the rotated part of every head of q [T][H][dnp + drp].  grid T
template <class T>
__global__ __launch_bounds__(256) void k_rope_inplace(T* q, const float2* rope, int H, int dnp, int drp, int dims, PassTabs p) {
  const int t = blockIdx.x, half = dims >> 1;
  const float2* rr = rope + (size_t)p.pos[t] * half;
  for (int i = threadIdx.x; i < H * half; i += 256) {
    const int h = i / half, j = i - h * half;
    T* v = q + ((size_t)t * H + h) * (dnp + drp) + dnp + 2 * j;
    const float2 cs = rr[j];
    const float u = (float)v[0], w = (float)v[1];
    v[0] = (T)(u * cs.x - w * cs.y);
    v[1] = (T)(w * cs.x + u * cs.y);
  }
}

static inline bool exp_supported(int dnp, int drp, int dvp) {
  return dnp + drp <= 256 && dnp >= 64 && dnp <= 192 && (drp == 64 || drp == 128) && (dvp == 64 || dvp == 128);
}
template <class T>
int exp_attn_launch(hipStream_t s, const ExpArgs& a) {
#ifndef KH_EXP_MR
#define KH_EXP_MR 1
#endif
  constexpr int MR = sizeof(T) == 2 ? KH_EXP_MR : 1;
  const size_t stage = (size_t)4 * Tile<T>::N * (a.dnp + a.drp) * sizeof(T) + (size_t)a.dvp * 64, lds = KH_EXP_STAGES * stage;
  auto go = [&](auto kern) -> int {
    if (lds > 64 * 1024) {
      const hipError_t e = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      if (e != hipSuccess) return (int)e;
    }
    hipLaunchKernelGGL(kern, dim3(a.H, (a.n + 64 * MR - 1) / (64 * MR)), dim3(256), lds, s, a);
    return KH_OK;
  };
  auto val = [&](auto kv) -> int {
    constexpr int KV = decltype(kv)::value;
    const int kn = a.dnp / 64, kr = a.drp / 64;
    if (kr == 1) {
      if (kn == 1) return go(k_expanded_attn<T, 1, 1, KV, MR>);
      if (kn == 2) return go(k_expanded_attn<T, 2, 1, KV, MR>);
      if (kn == 3) return go(k_expanded_attn<T, 3, 1, KV, MR>);
    } else if (kr == 2) {
      if (kn == 1) return go(k_expanded_attn<T, 1, 2, KV, MR>);
      if (kn == 2) return go(k_expanded_attn<T, 2, 2, KV, MR>);
    }
    return KH_ERR_UNSUPPORTED;
  };
  if (a.dvp == 64) return val(std::integral_constant<int, 1>());
  if (a.dvp == 128) return val(std::integral_constant<int, 2>());
  return KH_ERR_UNSUPPORTED;
}
}  // namespace khm
