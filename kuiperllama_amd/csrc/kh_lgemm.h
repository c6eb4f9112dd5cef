// kh_lgemm.h — GEMM of the layer-list models on the matrix cores: out[token][feature] = X[token][K] . W[feature][K],
// storage type T = bf16 or fp32 on both sides (kh_tile.h), fp32 accumulation.
//
//   * One workgroup = 4 waves (2 x 2) = a BM-token x BN-feature tile; K advances 128 bytes per stage through a ring
//     of NSTAGE LDS stages filled by the LDS-DMA path (global_load_lds_dwordx4): no staging registers, and
//     NSTAGE - 1 stages are in flight while one is multiplied.  The big tiles use two stages, which leaves room for
//     two workgroups per CU: one multiplies while the other waits (128 x 128: 0.43 - 0.50 of the bf16 peak, against
//     0.28 - 0.33 with three stages and one workgroup).
//   * LDS rows are 128 bytes.  Chunk c (16 bytes) of row r sits in slot c ^ (r & 7): the lanes of a fragment read
//     (16 rows, same chunk) touch all 64 banks.  The DMA writes slots in lane order, so the permutation is applied
//     to the GLOBAL address each lane requests.
//   * Weights are the first MFMA operand: a lane ends with four consecutive features of one token, which is what
//     every epilogue stores.
//   * Every row length is padded to KH_LPAD elements at load (zero weights), so K needs no tail; token and feature
//     tails are clamped on load and masked on store.
//   * Grouped form (experts): a device-side tile list maps blockIdx.y to (expert, first row, rows); the rows of X are
//     gathered through an index list.  Batched form (heads): blockIdx.z strides.
#pragma once
#include <vector>

#include "kh_q8ring.h"
#include "kh_tile.h"

#define KH_LPAD 64  // K granule of every weight row, in elements (128 bytes of bf16, 256 of fp32)

namespace khm {

enum LgEpi {
  LG_T = 0,        // out T (+ bias)
  LG_F32 = 1,      // out fp32 (+ bias)
  LG_SOFTPLUS = 2, // out fp32 = softplus(acc + bias[feature])
  LG_GATED = 3,    // weight rows come as 16 gate rows, 16 up rows, ...: out T = the gated unit, half the features
  LG_SPLIT = 4,    // features [0, n_split) -> out T, the rest -> out2 fp32
  LG_SOFTCAP = 5,  // out fp32 = cap * tanh(acc / cap); cap 0: plain
};

struct LgTile {  // one token tile of a grouped launch
  int group, row0, rows, pad;
};

struct LgArgs {
  const void* W;        // [N][ldw]
  const void* X;        // [M][ldx]
  void* out;            // [M][ldo]
  float* out2;          // LG_SPLIT: [M][ldo2]
  const float* bias;    // LG_SOFTPLUS; LG_T / LG_F32: optional
  const int32_t* gather;   // row of X for row m (grouped, optional)
  const LgTile* tiles;     // grouped launch
  const int32_t* n_tiles;  // number of valid entries of tiles
  size_t w_group;       // grouped: elements between the weights of two groups
  size_t w_z, x_z, o_z; // batched: elements per blockIdx.z
  int M, N, K, ldw, ldx, ldo, ldo2, n_split;
  float cap;
  GateAct act;          // LG_GATED
};

template <class T, int BM, int BN>
struct LgCfg {
  static constexpr int NSTAGE = BM + BN >= 192 ? 2 : (BM + BN >= 128 ? 3 : 4);
  static constexpr int STAGE = (BM + BN) * 128;
  static constexpr int LDS = NSTAGE * STAGE;
};

#pragma clang diagnostic push
#pragma clang diagnostic ignored "-Winline-asm"
// 64 lanes x 16 B from (base + voff[lane]) to LDS [dst + 16 lane], default cache policy
__device__ __forceinline__ void dma_x4_keep(const void* base, unsigned voff, unsigned dst) {
  asm volatile("s_mov_b32 m0, %2\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %0, %1"
               :
               : "v"(voff), "s"(base), "s"(dst)
               : "memory", "m0");
}
#pragma clang diagnostic pop

template <class T, int BM, int BN, int EPI>
__global__ __launch_bounds__(256) void k_lgemm(const LgArgs a) {
  typedef Tile<T> TL;
  typedef typename TL::frag frag;
  constexpr int NST = LgCfg<T, BM, BN>::NSTAGE, STAGE = LgCfg<T, BM, BN>::STAGE;
  constexpr int TM = BM / 32, TN = BN / 32;  // 16-wide tiles per wave: tokens, features
  constexpr int NL = (BM + BN) / 32;         // LDS-DMA requests per wave and stage
  extern __shared__ __attribute__((aligned(1024))) char smem_raw[];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const char* W = (const char*)a.W;
  const char* X = (const char*)a.X;
  int m_lo = 0, m_n = a.M;  // rows [m_lo, m_lo + m_n) of the row index space belong to this launch / group
  int mt0;                  // first row of the tile
  if (a.tiles) {
    if ((int)blockIdx.y >= *a.n_tiles) return;  // uniform: the grid is an upper bound
    const LgTile t = a.tiles[blockIdx.y];
    W += (size_t)t.group * a.w_group * sizeof(T);
    m_lo = t.row0;
    m_n = t.rows;
    mt0 = t.row0;
  } else {
    mt0 = (int)blockIdx.y * BM;
  }
  W += (size_t)blockIdx.z * a.w_z * sizeof(T);
  X += (size_t)blockIdx.z * a.x_z * sizeof(T);
  const int f0 = (int)blockIdx.x * BN;
  const int m_last = m_lo + m_n - 1;
  // ---- staging addresses: request j of wave w covers rows 8 (4 j + w) .. +8 of the stacked (tokens, features) tile
  unsigned voff[NL];
  const int sub = lane >> 3, ch = (lane & 7) ^ sub;
#pragma unroll
  for (int j = 0; j < NL; ++j) {
    const int r = 8 * (4 * j + wave) + sub;
    if (j < BM / 32) {
      int m = mt0 + r;
      m = m < m_last ? m : m_last;
      const int row = a.gather ? a.gather[m] : m;
      voff[j] = (unsigned)row * (unsigned)(a.ldx * (int)sizeof(T)) + 16u * ch;
    } else {
      int f = f0 + r - BM;
      f = f < a.N ? f : a.N - 1;
      voff[j] = (unsigned)f * (unsigned)(a.ldw * (int)sizeof(T)) + 16u * ch;
    }
  }
  const unsigned lds0 = (unsigned)__builtin_amdgcn_readfirstlane((int)kh_lds_addr(smem_raw)) + 1024u * wave;
  auto issue = [&](int slot) __attribute__((always_inline)) {
#pragma unroll
    for (int j = 0; j < NL; ++j) {
      dma_x4_keep(j < BM / 32 ? (const void*)X : (const void*)W, voff[j], lds0 + (unsigned)(slot * STAGE + j * 4096));
      voff[j] += 128;
    }
  };
  const int nk = a.K * (int)sizeof(T) / 128;  // stages
  f32x4 acc[TN][TM];
#pragma unroll
  for (int n = 0; n < TN; ++n)
#pragma unroll
    for (int m = 0; m < TM; ++m) acc[n][m] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < NST - 1; ++s)
    if (s < nk) issue(s);
  const int wm = wave & 1, wn = wave >> 1;
  const int fr = lane & 15, fh = lane >> 4;
  int slot = 0, fill = NST - 1;
  for (int k = 0; k < nk; ++k) {
    // stage k has landed when at most the requests of the stages behind it are outstanding
    if (k + NST - 2 < nk) wait_vm<(NST - 2) * NL>();
    else wait_vm<0>();
    __syncthreads();
    if (k + NST - 1 < nk) issue(fill);
    const char* st = smem_raw + slot * STAGE;
    // both halves of the stage are requested from LDS before the first product: the second half arrives under the
    // products of the first (left to itself the compiler reads one half at a time; 0.40 -> 0.43 ... 0.50 of the peak)
    frag fx[2][TM], fw[2][TN];
#pragma unroll
    for (int b = 0; b < 2; ++b) {
#pragma unroll
      for (int m = 0; m < TM; ++m) {
        const int r = wm * (BM / 2) + m * 16 + fr;
        fx[b][m] = *(const frag*)(st + r * 128 + (((4 * b + fh) ^ (r & 7)) << 4));
      }
#pragma unroll
      for (int n = 0; n < TN; ++n) {
        const int r = BM + wn * (BN / 2) + n * 16 + fr;
        fw[b][n] = *(const frag*)(st + r * 128 + (((4 * b + fh) ^ (r & 7)) << 4));
      }
    }
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int n = 0; n < TN; ++n)
#pragma unroll
        for (int m = 0; m < TM; ++m) acc[n][m] = TL::mma(fw[b][n], fx[b][m], acc[n][m]);
    slot = slot + 1 == NST ? 0 : slot + 1;
    fill = fill + 1 == NST ? 0 : fill + 1;
  }
  // ---- epilogue: lane (fr, fh) of tile (n, m): token mt0 + .. + fr, features f .. f + 3
#pragma unroll
  for (int m = 0; m < TM; ++m) {
    const int tok = mt0 + wm * (BM / 2) + m * 16 + fr;
    if (tok > m_last) continue;
    if (EPI == LG_GATED) {
#pragma unroll
      for (int n = 0; n + 1 < TN; n += 2) {
        const int f = f0 + wn * (BN / 2) + n * 16;  // a multiple of 32: gate tile; the up tile follows
        const int c = (f >> 1) + 4 * fh;
        f32x4 v;
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = gated1(a.act, acc[n][m][i], acc[n + 1][m][i]);
        if (f < a.N) *(typename TL::quad*)((T*)a.out + (size_t)tok * a.ldo + c) = to_quad<T>(v);
      }
    } else {
#pragma unroll
      for (int n = 0; n < TN; ++n) {
        const int f = f0 + wn * (BN / 2) + n * 16 + 4 * fh;
        f32x4 v = acc[n][m];
        if ((EPI == LG_T || EPI == LG_F32) && a.bias) {
#pragma unroll
          for (int i = 0; i < 4; ++i) v[i] += a.bias[f + i < a.N ? f + i : 0];
        }
        if (EPI == LG_T) {
          T* o = (T*)a.out + (size_t)blockIdx.z * a.o_z + (size_t)tok * a.ldo + f;
          if (f + 3 < a.N && (a.ldo & 3) == 0) {
            *(typename TL::quad*)o = to_quad<T>(v);
          } else {
#pragma unroll
            for (int i = 0; i < 4; ++i)
              if (f + i < a.N) o[i] = (T)v[i];
          }
        } else {
          f32x4 y = v;
          if (EPI == LG_SOFTPLUS) {
#pragma unroll
            for (int i = 0; i < 4; ++i) y[i] = softplus1(v[i] + a.bias[f + i < a.N ? f + i : 0]);
          } else if (EPI == LG_SOFTCAP) {
#pragma unroll
            for (int i = 0; i < 4; ++i) y[i] = a.cap > 0.f ? a.cap * tanhf(v[i] / a.cap) : v[i];
          }
          // destination of the four features: one array, unless they straddle LG_SPLIT's border
          const bool to_t = EPI == LG_SPLIT && f + 3 < a.n_split, cut = EPI == LG_SPLIT && !to_t && f < a.n_split;
          float* o = EPI == LG_SPLIT ? a.out2 + (size_t)tok * a.ldo2 + (f - a.n_split) : (float*)a.out + (size_t)tok * a.ldo + f;
          const int ld = EPI == LG_SPLIT ? a.ldo2 : a.ldo;
          if (to_t) {
            T* ot = (T*)a.out + (size_t)tok * a.ldo + f;
#pragma unroll
            for (int i = 0; i < 4; ++i) ot[i] = (T)y[i];
          } else if (!cut && f + 3 < a.N && (ld & 3) == 0) {
            *(f32x4*)o = y;
          } else {
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              if (f + i >= a.N) continue;
              if (EPI == LG_SPLIT && f + i < a.n_split) ((T*)a.out)[(size_t)tok * a.ldo + f + i] = (T)y[i];
              else o[i] = y[i];
            }
          }
        }
      }
    }
  }
}

// Tile choice.  Plain / batched launches: the largest tile that still gives the chip enough workgroups (one per CU is
// not: nobody covers its barriers).  Grouped
// launches: BM = the row granule the tile list was built with (lg_group_bm).
static inline int lg_group_bm(long rows, int groups) {
  const long per = rows / (groups > 0 ? groups : 1);
  return per > 64 ? 128 : (per > 24 ? 64 : 32);
}
template <class T, int EPI>
int lg_launch(hipStream_t s, const LgArgs& a, int zdim = 1, int group_bm = 0, int max_tiles = 0) {
  auto go = [&](auto kern, int BM, int BN, int lds) -> int {
    if (lds > 64 * 1024) {  // the dynamic-LDS opt-in is per (device, kernel): once
      struct Done { int dev; const void* fn; };
      static thread_local std::vector<Done> done;
      int dev = 0;
      (void)hipGetDevice(&dev);
      bool hit = false;
      for (const auto& d : done) hit = hit || (d.dev == dev && d.fn == (const void*)kern);
      if (!hit) {
        const hipError_t e = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds);
        if (e != hipSuccess) return (int)e;
        done.push_back({dev, (const void*)kern});
      }
    }
    const int gy = a.tiles ? max_tiles : (a.M + BM - 1) / BM;
    hipLaunchKernelGGL(kern, dim3((a.N + BN - 1) / BN, gy, zdim), dim3(256), lds, s, a);
    return KH_OK;
  };
  auto tiles = [&](int BM, int BN) { return (long)((a.N + BN - 1) / BN) * ((a.M + BM - 1) / BM) * zdim; };
  if (a.tiles ? group_bm == 128 : a.M > 64 && tiles(128, 128) >= 400)
    return go(k_lgemm<T, 128, 128, EPI>, 128, 128, LgCfg<T, 128, 128>::LDS);
  if (a.tiles ? group_bm == 32 : a.M <= 32) return go(k_lgemm<T, 32, 64, EPI>, 32, 64, LgCfg<T, 32, 64>::LDS);
  if (a.tiles || tiles(64, 128) >= 400) return go(k_lgemm<T, 64, 128, EPI>, 64, 128, LgCfg<T, 64, 128>::LDS);
  return go(k_lgemm<T, 64, 64, EPI>, 64, 64, LgCfg<T, 64, 64>::LDS);
}
}  // namespace khm
