// kh_hybrid_step.hip — layer-list models: the decode step of the generate loop, sequence slots, batches.
#include <string.h>

#include <algorithm>
#include <type_traits>

#include "kh_fused.h"
#include "kh_hybrid.h"
#include "kh_ldecode.h"

using namespace khm;

namespace khm {
// buffers and launch plan of the fused decode step for up to KH_HY_DECODE_B sequences
struct Hybrid::Step {
  int bmax = 0;  // sequences one fused step can take (0: the geometry does not fit; everything runs as passes)
  float *x[3] = {nullptr, nullptr, nullptr}, *xn2 = nullptr, *in = nullptr, *xc = nullptr, *mid = nullptr, *v = nullptr,
        *he = nullptr, *hs = nullptr, *z = nullptr, *id_w = nullptr, *sh_g = nullptr, *part = nullptr, *logits = nullptr;
  void* Q = nullptr;
  int32_t *ids = nullptr, *tabs = nullptr;
  int32_t* h_tabs = nullptr;
  int nsplit = 1, head_wg = 1;
  ~Step() {
    for (void* p : {(void*)x[0], (void*)x[1], (void*)x[2], (void*)xn2, (void*)in, (void*)xc, (void*)mid, (void*)v, (void*)he,
                    (void*)hs, (void*)z, (void*)id_w, (void*)sh_g, (void*)part, (void*)logits, Q, (void*)ids, (void*)tabs})
      if (p) (void)hipFree(p);
    if (h_tabs) (void)hipHostFree(h_tabs);
  }
};
Hybrid::Hybrid() {}
Hybrid::~Hybrid() {}

namespace {
constexpr int kMaxLds = 160 * 1024;
// tabs: tok[B], pos[B], slot[B] (uploaded per batch) at 0, B, 2B of KH_HY_DECODE_B; zeros behind them
enum { TB_TOK = 0, TB_POS = KH_HY_DECODE_B, TB_SLOT = 2 * KH_HY_DECODE_B, TB_ZERO = 3 * KH_HY_DECODE_B,
       TB_N = 4 * KH_HY_DECODE_B };

template <class T>
size_t vec_b(int n) { return Ld<T>::vec_bytes(n); }
template <class T>
size_t lds_out(const Hybrid& hy, const HyLayer& l, int B) {
  const int nbv = Ld<T>::blocks(l.out_mat().ld);
  const int nf = l.ff.on ? l.ff.top * Ld<T>::blocks(l.ff.ffp) + (l.ff.sffp ? Ld<T>::blocks(l.ff.sffp) : 0) : 0;
  (void)hy;
  return ((size_t)B * nbv + nf) * Ld<T>::BE * 4;
}
template <class T>
bool fits(const Hybrid& hy, int B) {
  const size_t room = kMaxLds - 2048;  // static shared memory of the kernels
  if (hy.c.widthp > 8192 || B * vec_b<T>(hy.c.widthp) > room) return false;
  if (hy.enter.N && B * vec_b<T>(hy.enter.ld) > room) return false;
  for (auto& l : hy.layers) {
    if (lds_out<T>(hy, l, B) > room) return false;
    if (l.mixer == HY_MAMBA1 && B * vec_b<T>(l.mb.innerp) > room) return false;
    if (l.mixer == HY_LATENT && (B * vec_b<T>(l.la.qrp) > room)) return false;
  }
  return true;
}

template <class K, class... A>
int go(K kern, dim3 grid, int wg, size_t lds, hipStream_t s, A... args) {
  if (lds > 64 * 1024) {
    struct Done { int dev; const void* fn; size_t lds; };
    static thread_local std::vector<Done> done;
    int dev = 0;
    (void)hipGetDevice(&dev);
    bool hit = false;
    for (const auto& d : done) hit = hit || (d.dev == dev && d.fn == (const void*)kern && d.lds >= lds);
    if (!hit) {
      const hipError_t e = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      if (e != hipSuccess) return (int)e;
      done.push_back({dev, (const void*)kern, lds});
    }
  }
  hipLaunchKernelGGL(kern, grid, dim3(wg), lds, s, args...);
  return KH_OK;
}
#define TRY(e)                    \
  do {                            \
    const int _rc = (e);          \
    if (_rc != KH_OK) return _rc; \
  } while (0)

int cdiv(int a, int b) { return (a + b - 1) / b; }

template <class T>
int launch_scan(const LdScanArgs& a, int B, hipStream_t s) {
  const dim3 grid(cdiv(a.C, 16), B);
  if (a.N <= 16) return go(k_ld_scan<T, 1>, grid, 256, 0, s, a);
  if (a.N <= 32) return go(k_ld_scan<T, 2>, grid, 256, 0, s, a);
  if (a.N <= 64) return go(k_ld_scan<T, 4>, grid, 256, 0, s, a);
  if (a.N <= 128) return go(k_ld_scan<T, 8>, grid, 256, 0, s, a);
  return go(k_ld_scan<T, 16>, grid, 256, 0, s, a);
}
// staging depth (float4 per thread) that covers a padded row of the residual stream
template <class T, class F>
int with_nv(int ld, F&& f) {
  const int n = cdiv(Ld<T>::blocks(ld) * Ld<T>::BE / 4, 256);
  if (n <= 2) return f(std::integral_constant<int, 2>());
  if (n <= 4) return f(std::integral_constant<int, 4>());
  return f(std::integral_constant<int, 8>());
}
template <class F>
int with_rp(int n_out, F&& f) {
  const int per = moe_per(n_out);
  if (per == 1) return f(std::integral_constant<int, 1>());
  if (per == 4) return f(std::integral_constant<int, 4>());
  return f(std::integral_constant<int, 16>());
}

// waves of a row pair over nblk blocks (k_ld_out, k_ld_enter): as many as keep each wave's share within its two tiles and
// give every CU a workgroup, while the launch has at most four per CU
int split_waves(int rows, int nblk) {
  int ks = 1;
  while (ks < 8 && nblk >= 2 * ks && (nblk / ks > 8 || cdiv(cdiv(rows, 2) * ks, 8) < 256) && cdiv(cdiv(rows, 2) * ks * 2, 8) <= 1024)
    ks *= 2;
  return ks;
}

// One token of B sequences: tables at (tok, pos, slot); logits to `logits` [B][V]; argmax partials of sequence 0 to
// the model's sampler buffers.
template <class T, int B>
int step(kh_model* m, const LdTabs tb, float* logits) {
  Hybrid& hy = *m->hy;
  Hybrid::Step& st = *hy.step_st;
  hipStream_t s = m->stream;
  const int W = hy.c.width, Wp = hy.c.widthp;
  float* x_in = st.x[0];
  for (size_t ri = 0; ri < hy.runs.size(); ++ri) {
    const HyRun& r = hy.runs[ri];
    const HyLayer& l = hy.layers[(size_t)r.layer];
    const HyMoe& f = l.ff;
    const HyHeads& ha = l.ha;
    const bool mamba = l.mixer == HY_MAMBA1, heads = l.mixer == HY_HEADS, through = r.pass >= 0 && hy.enter.N;
    const bool changed = !through && (ri == 0 || r.pass >= 0);
    float* x_cur = through || changed ? st.x[2] : x_in;
    float* x_out = x_in == st.x[0] ? st.x[1] : st.x[0];
    const HyMat& w_in = mamba ? l.mb.in : (heads ? ha.qkvg : l.la.dqkv);
    const int in_ld = w_in.N;
    const LdEmbed emb{hy.embed.w, hy.pos_emb.w, hy.c.emb_scale};
    if (through) {
      LdEnterArgs a{hy.enter.w, ri == 0 ? nullptr : x_in, st.x[2], emb, W, Wp, 1, tb};
      a.ks = split_waves(W, Ld<T>::blocks(hy.enter.ld));
      TRY(go(k_ld_enter<T, B>, dim3(cdiv(cdiv(W, 2) * a.ks, 8)), 512, B * vec_b<T>(hy.enter.ld), s, a));
    }
    {
      LdInArgs a{};
      auto seg = [&](const HyMat& w, float* out, int rows, int ldo, int kind, int norm2) {
        LdInSeg& g = a.seg[a.nseg++];
        g.w = w.w;
        g.out = out;
        g.rows = rows;
        g.ldo = ldo;
        g.kind = kind;
        g.norm2 = norm2;
      };
      seg(w_in, st.in, in_ld, in_ld, mamba ? LDI_CONV : LDI_PLAIN, 0);
      if (heads) a.seg[0].bias = ha.qkvg_b.p;
      if (f.top) seg(f.zr, st.z, f.zr.N, f.zr.N, LDI_PLAIN, 1);
      if (f.sff) seg(f.sgu, st.hs, f.sffp, f.sffp, LDI_GATED, 1);
      a.act = f.sact;
      int total = 0, wg = 0;
      auto items = [&](const LdInSeg& g) { return cdiv(g.rows, g.kind == LDI_GATED ? 2 : 4); };
      for (int i = 0; i < a.nseg; ++i) total += items(a.seg[i]);
      const int ipw = cdiv(total, 2048);
      for (int i = 0; i < a.nseg; ++i) {
        a.seg[i].wg0 = wg;
        a.seg[i].nwg = cdiv(items(a.seg[i]), 4 * ipw);
        wg += a.seg[i].nwg;
      }
      a.x_in = through ? x_cur : x_in;
      a.x_cur = changed ? x_cur : nullptr;
      a.emb = emb;
      a.step = r.pass >= 0 && hy.step.on ? hy.step.p + (size_t)r.pass * Wp : nullptr;
      a.w1 = l.n1.p;
      a.b1 = l.n1b.p;
      a.w2 = l.norm2().p;
      a.b2 = l.norm2_b().p;
      a.xn2 = f.top ? st.xn2 : nullptr;
      a.W = W;
      a.ld = Wp;
      a.from_embed = ri == 0 && !through;
      a.add_x0 = r.pass > 0 && !through;
      a.rms = hy.c.rms;
      a.eps = hy.c.eps;
      a.t = tb;
      if (mamba) {
        a.conv_w = l.mb.conv.p;
        a.conv_b = l.mb.conv_b.p;
        a.conv_st = hy.state + r.conv_off;
        a.slot_stride = hy.st_slot;
        a.xc = st.xc;
        a.inner = l.mb.inner;
        a.taps = l.mb.taps;
        a.xc_ld = l.mb.innerp;
      }
      TRY(with_nv<T>(Wp, [&](auto nv) { return go(k_ld_in<T, B, decltype(nv)::value>, dim3(wg), 256, B * vec_b<T>(Wp), s, a); }));
    }
    {
      LdMidArgs a{};
      a.t = tb;
      a.eps = hy.c.eps;
      size_t lds = 0;
      if (f.top) {
        a.z = st.z;
        a.corr = f.corr.p;
        a.xn2 = st.xn2;
        a.gu = f.gu.w;
        a.he = st.he;
        a.ids = st.ids;
        a.id_w = st.id_w;
        a.sh_g = st.sh_g;
        a.top = f.top;
        a.n_out = f.n_out();
        a.n_expert = f.E;
        a.shared = f.sgate;
        a.over_chosen = f.over_chosen;
        a.act = f.act;
        a.ffp = f.ffp;
        a.ldz = f.zr.N;
        a.W = W;
        a.ldw = f.gu.ld;
        a.nwg_e = cdiv(f.ffp / 2, 4 * cdiv(B * f.top * f.ffp / 2, 3072));
        lds = vec_b<T>(Wp);
      }
      a.ldv = mamba ? l.mb.innerp : in_ld;
      int extra = 0;
      if (heads) {
        extra = cdiv(B * ha.G, 4);
        a.heads = 1;
        a.hr = ha.head_row(hy.c.eps);
        a.raw = st.in;
        a.cache = (T*)m->kcache + r.kv_off;
        a.slot_elems = hy.kv_slot;
      } else {
        const HyMat& wm = mamba ? l.mb.x : l.la.uq;
        a.wm = wm.w;
        a.rows = wm.N;
        a.ldm = wm.ld;
        a.n = mamba ? l.mb.inner : l.la.qr;
        a.n4 = l.mb.innerp / 4;  // convolved inputs are padded with zeros
        a.v = mamba ? st.xc : st.in;
        a.vnorm = mamba ? nullptr : l.la.qn.p;
        a.om = st.mid;
        a.ldo = wm.N;
        a.nwg_m = std::min(cdiv(cdiv(wm.N, 4), 4), 512);
        lds = std::max(lds, B * vec_b<T>(wm.ld));
      }
      if (l.mixer == HY_LATENT) {
        const HyLatent& la = l.la;
        extra = B;
        a.latent = 1;
        a.raw = st.in;
        a.kvn = la.kvn.p;
        a.rope = la.rope;
        a.cache = (T*)m->kcache + r.kv_off;
        a.slot_elems = hy.kv_slot;
        a.qr = la.qr;
        a.R = la.R;
        a.dr = la.dr;
        a.Rp = la.Rp;
        a.row = la.row();
        a.dims = la.dims;
      }
      TRY(with_nv<T>(Wp, [&](auto nv) {
        return with_rp(f.top ? f.n_out() : 1, [&](auto rp) {
          return go(k_ld_mid<T, B, decltype(nv)::value, decltype(rp)::value>, dim3(B * a.top * a.nwg_e + a.nwg_m + extra), 256, lds,
                    s, a);
        });
      }));
    }
    if (mamba) {
      const HyMamba& mb = l.mb;
      LdScanArgs a{st.xc, st.in, st.mid, mb.dt.w, mb.dt_b.p, mb.A2.p, mb.D.p, hy.state + r.st_off, st.v, hy.st_slot,
                   mb.inner, mb.state, mb.rankp, mb.innerp, mb.innerp, tb};
      TRY(launch_scan<T>(a, B, s));
    } else if (heads) {
      HeadsArgs a = heads_args(hy, ha, (const T*)m->kcache + r.kv_off);
      a.raw = st.in;
      a.raw_f32 = 1;
      a.ldr = in_ld;
      a.part = st.part;
      a.nsplit = ha.nsplit;
      a.p.seg_slot = tb.slot;
      a.p.seg_pos0 = tb.pos;
      TRY(heads_attn_launch<T>(s, a, B * cdiv(ha.H / ha.G, 16), 16));
      LdMergeArgs mg{st.part, ha.gate ? st.in + ha.g_off() : nullptr, st.v, ha.H, ha.nsplit, ha.dvp, ha.dvr, in_ld, ha.o.ld,
                     ha.span, tb.pos};
      TRY(go(k_ld_merge, dim3(ha.H, B), 256, 256 * 16, s, mg));
    } else {
      const HyLatent& la = l.la;
      LdAbsorbArgs ab{st.mid, la.ukT.w, la.rope, st.Q, la.H, std::max(1, std::min(cdiv(la.Rp, 32), cdiv(512, la.H * B))),
                      la.dnp, la.dr, la.drp, la.Rp, la.row(), la.dims, tb};
      TRY(go(k_ld_absorb<T>, dim3(la.H * ab.nwg, B), 256, (size_t)la.dnp * 4, s, ab));
      const int cp = la.H <= 32 ? 4 : (la.Rp > 256 ? 2 : 1), tiles = B * cdiv(la.H, 64 / cp);
      LatArgs at{};
      at.Q = st.Q;
      at.cache = (const T*)m->kcache + r.kv_off;
      at.slot_elems = hy.kv_slot;
      at.sink = la.sink.p;
      at.part = st.part;
      at.H = la.H;
      at.Rp = la.Rp;
      at.row = la.row();
      at.nsplit = st.nsplit;
      at.scale2 = la.scale * 1.44269504088896f;
      at.p.seg_slot = tb.slot;
      at.p.seg_pos0 = tb.pos;
      TRY(lat_attn_launch<T>(s, at, tiles, cp));
      LdValuesArgs va{st.part, la.uv.w, st.v, la.H, std::max(1, std::min(cdiv(la.dvp, 16), cdiv(128, la.H * B))), st.nsplit,
                      la.Rp, la.dvp, tb.pos};
      TRY(go(k_ld_values<T>, dim3(la.H * va.nwg, B), 256, vec_b<T>(la.Rp) + 256 * 16 + (size_t)la.Rp * 4, s, va));
    }
    {
      const HyMat& wo = l.out_mat();
      LdOutArgs a{};
      a.wo = wo.w;
      a.v = st.v;
      a.n4v = wo.ld / 4;
      a.ld = Wp;
      a.ld_v = wo.ld;
      a.ldv = wo.ld;
      a.bias = heads ? ha.o_b.p : nullptr;
      a.mult = hy.c.mult;
      a.x_cur = x_cur;
      a.x_out = x_out;
      a.W = W;
      if (f.on) {
        a.moe = 1;
        a.down = f.down.w;
        a.sdown = f.sdown.w;
        a.he = st.he;
        a.hs = st.hs;
        a.ids = st.ids;
        a.id_w = f.ident ? st.id_w : nullptr;
        a.sh_g = f.sgate ? st.sh_g : nullptr;
        a.xn2 = st.xn2;
        a.top = f.top;
        a.ffp = f.ffp;
        a.sffp = f.sffp;
      }
      a.ks = split_waves(W, Ld<T>::blocks(wo.ld) + (f.on ? f.top * Ld<T>::blocks(f.ffp) + (f.sff ? Ld<T>::blocks(f.sffp) : 0) : 0));
      TRY(go(k_ld_out<T, B>, dim3(cdiv(cdiv(W, 2) * a.ks, 8)), 512, lds_out<T>(hy, l, B), s, a));
    }
    x_in = x_out;
  }
  LdHeadArgs h{x_in, hy.fnorm.p, hy.fnorm_b.p, hy.head.w, logits, m->part_val, m->part_idx, W, Wp, hy.c.vocab, hy.c.rms, hy.c.eps,
               hy.c.cap};
  return with_nv<T>(Wp, [&](auto nv) { return go(k_ld_head<T, B, decltype(nv)::value>, dim3(st.head_wg), 256, B * vec_b<T>(Wp), s, h); });
}
template <class T>
int step_b(kh_model* m, int B, const LdTabs& tb, float* logits) {
  if (B == 1) return step<T, 1>(m, tb, logits);
  if (B == 2) return step<T, 2>(m, tb, logits);
  return step<T, 4>(m, tb, logits);
}
int step_any(kh_model* m, int B, const LdTabs& tb, float* logits) {
  return m->hy->f32 ? step_b<float>(m, B, tb, logits) : step_b<bf16>(m, B, tb, logits);
}
}  // namespace

int hy_step_init(kh_model* m) {
  Hybrid& hy = *m->hy;
  hy.step_st.reset(new Hybrid::Step());
  Hybrid::Step& st = *hy.step_st;
  for (int B : {1, 2, 4})
    if (hy.f32 ? fits<float>(hy, B) : fits<bf16>(hy, B)) st.bmax = B;
  const size_t B = KH_HY_DECODE_B, W = (size_t)hy.c.widthp;
  size_t in = 1, xc = 1, mid = 1, v = 1, he = 1, hs = 1, z = 1, top = 1, Q = 1, part = 1, hpart = 1;
  auto up = [](size_t& a, size_t n) { a = a > n ? a : n; };
  for (auto& l : hy.layers) {
    if (l.mixer == HY_MAMBA1) {
      up(in, 2 * (size_t)l.mb.inner);
      up(xc, (size_t)l.mb.innerp);
      up(mid, (size_t)l.mb.x.N);
      up(v, (size_t)l.mb.innerp);
    } else if (l.mixer == HY_HEADS) {
      up(in, (size_t)l.ha.qkvg.N);
      up(v, (size_t)l.ha.o.ld);
      up(hpart, (size_t)l.ha.H * (l.ha.dvp + 4) * l.ha.nsplit);
    } else {
      up(in, (size_t)l.la.dqkv.N);
      up(mid, (size_t)l.la.uq.N);
      up(v, (size_t)l.la.H * l.la.dvp);
      up(Q, (size_t)l.la.H * l.la.row());
      up(part, (size_t)l.la.H * (l.la.Rp + 4));
    }
    if (l.ff.on) {
      up(he, (size_t)l.ff.top * l.ff.ffp);
      up(hs, (size_t)l.ff.sffp);
      up(z, (size_t)l.ff.zr.N);
      up(top, (size_t)l.ff.top);
    }
  }
  // time splits: about one workgroup per CU over the row tiles of one sequence
  st.nsplit = 2;
  while (st.nsplit < 128 && st.nsplit * KH_LAT_SPLIT_MIN < m->cfg.cache_len) st.nsplit *= 2;
  auto f = [&](float** p, size_t n) -> int {
    TRY(dalloc(p, n));
    return (int)hipMemsetAsync(*p, 0, n * 4, m->stream);
  };
  for (float** p : {&st.x[0], &st.x[1], &st.x[2], &st.xn2}) TRY(f(p, B * W));
  TRY(f(&st.in, B * in));
  TRY(f(&st.xc, B * xc));
  TRY(f(&st.mid, B * mid));
  TRY(f(&st.v, B * v));
  TRY(f(&st.he, B * he));
  TRY(f(&st.hs, B * hs));
  TRY(f(&st.z, B * z));
  TRY(f(&st.id_w, B));
  TRY(f(&st.sh_g, B));
  TRY(f(&st.part, B * std::max(part * (size_t)st.nsplit, hpart)));
  TRY(f(&st.logits, B * (size_t)hy.c.vocab));
  TRY(f((float**)&st.Q, B * Q));
  TRY(dalloc(&st.ids, B * top));
  TRY(dalloc(&st.tabs, TB_N));
  KH_CHECK_HIP(hipHostMalloc((void**)&st.h_tabs, TB_N * 4, hipHostMallocDefault));
  memset(st.h_tabs, 0, TB_N * 4);
  KH_CHECK_HIP(hipMemcpyAsync(st.tabs, st.h_tabs, TB_N * 4, hipMemcpyHostToDevice, m->stream));
  st.head_wg = std::min(cdiv(cdiv(hy.c.vocab, 4), 4), 1024);
  m->nparts = st.head_wg;
  TRY(dalloc(&m->part_val, (size_t)m->nparts));
  TRY(dalloc(&m->part_idx, (size_t)m->nparts));
  return KH_OK;
}

// the generate loop's step: (d_token, d_pos) of slot 0, sampler behind it
void hy_launch_step(kh_model* m, int advance, int n_forced) {
  Hybrid& hy = *m->hy;
  if (hy.step_st->bmax >= 1) {
    const LdTabs tb{m->d_token, m->d_pos, hy.step_st->tabs + TB_ZERO};
    (void)step_any(m, 1, tb, m->logits);
  } else {  // the pass kernels leave logits; the sampler wants partials
    (void)hy_unfused_step(m);
    (void)hy_argmax_partial(m);
  }
  launch_sample(m, advance, n_forced);
}
int hy_launches(const kh_model* m) {
  int n = 2;
  for (const HyRun& r : m->hy->runs) {
    const int mixer = m->hy->layers[(size_t)r.layer].mixer;
    n += mixer == HY_MAMBA1 ? 4 : (mixer == HY_LATENT ? 6 : 5);
    if (r.pass >= 0 && m->hy->enter.N) ++n;
  }
  return n;
}
int hy_decode_max(const kh_model* m) { return m->hy->step_st->bmax; }
// one token of each of n sequences (n <= hy_decode_max), logits [n][vocab] to the host
int hy_decode(kh_model* m, const HyEntry* e, int n, float* h_logits) {
  Hybrid& hy = *m->hy;
  Hybrid::Step& st = *hy.step_st;
  KH_CHECK_HIP(hipSetDevice(m->opts.device));
  KH_CHECK_HIP(hipStreamSynchronize(m->stream));  // the pinned table of the call before is free again
  for (int i = 0; i < n; ++i) {
    st.h_tabs[TB_TOK + i] = e[i].tok[0];
    st.h_tabs[TB_POS + i] = e[i].pos0;
    st.h_tabs[TB_SLOT + i] = e[i].slot;
  }
  KH_CHECK_HIP(hipMemcpyAsync(st.tabs, st.h_tabs, TB_ZERO * 4, hipMemcpyHostToDevice, m->stream));
  for (int i = 0; i < n;) {  // n = 3: 2 + 1
    const int B = n - i >= 4 ? 4 : (n - i >= 2 ? 2 : 1);
    const LdTabs tb{st.tabs + TB_TOK + i, st.tabs + TB_POS + i, st.tabs + TB_SLOT + i};
    TRY(step_any(m, B, tb, st.logits));
    if (h_logits)
      KH_CHECK_HIP(hipMemcpyAsync(h_logits + (size_t)i * hy.c.vocab, st.logits, (size_t)B * hy.c.vocab * 4,
                                  hipMemcpyDeviceToHost, m->stream));
    i += B;
  }
  TRY(kh_launch_status());
  if (h_logits) KH_CHECK_HIP(hipStreamSynchronize(m->stream));
  return KH_OK;
}
}  // namespace khm

// ---- sequences ---------------------------------------------------------------------------------------------------
extern "C" int kh_seq_open(kh_model* m, int32_t* seq) {
  if (!m || !seq) return KH_ERR_INVALID_ARG;
  std::vector<int>& len = m->hy ? m->hy->len : m->seq_len;
  if (!m->hy && len.empty()) len.assign(1, -1);
  for (size_t i = 0; i < len.size(); ++i)
    if (len[i] < 0) {
      len[i] = 0;
      *seq = (int32_t)i;
      return KH_OK;
    }
  return KH_ERR_RANGE;
}
extern "C" int kh_seq_close(kh_model* m, int32_t seq) {
  if (!m) return KH_ERR_INVALID_ARG;
  std::vector<int>& len = m->hy ? m->hy->len : m->seq_len;
  if (seq < 0 || seq >= (int)len.size() || len[(size_t)seq] < 0) return KH_ERR_RANGE;
  len[(size_t)seq] = -1;
  return KH_OK;
}
extern "C" int kh_seq_length(const kh_model* m, int32_t seq) {
  if (!m) return KH_ERR_INVALID_ARG;
  const std::vector<int>& len = m->hy ? m->hy->len : m->seq_len;
  return seq < 0 || seq >= (int)len.size() ? KH_ERR_RANGE : (len[(size_t)seq] < 0 ? KH_ERR_RANGE : len[(size_t)seq]);
}

namespace {
int forward_checks(const kh_model* m, const std::vector<int>& len, const kh_batch_entry* e, int n) {
  std::vector<char> seen(len.size(), 0);
  for (int i = 0; i < n; ++i) {
    if (e[i].seq < 0 || e[i].seq >= (int)len.size() || len[(size_t)e[i].seq] < 0) return KH_ERR_RANGE;
    if (seen[(size_t)e[i].seq]++) return KH_ERR_INVALID_ARG;
    if (e[i].n_tokens <= 0 || !e[i].tokens || e[i].n_want < 0 || (e[i].n_want > 0 && !e[i].want)) return KH_ERR_INVALID_ARG;
    if ((int64_t)len[(size_t)e[i].seq] + e[i].n_tokens > m->cfg.cache_len) return KH_ERR_RANGE;
    for (int k = 0; k < e[i].n_tokens; ++k)
      if (e[i].tokens[k] < 0 || e[i].tokens[k] >= m->cfg.vocab_size) return KH_ERR_RANGE;
    for (int k = 0; k < e[i].n_want; ++k)
      if (e[i].want[k] < 0 || e[i].want[k] >= e[i].n_tokens || (k && e[i].want[k] <= e[i].want[k - 1])) return KH_ERR_INVALID_ARG;
  }
  return KH_OK;
}

int forward_layers(kh_model* m, const kh_batch_entry* e, int n, float* h_logits) {
  Hybrid& hy = *m->hy;
  std::vector<HyEntry> es;
  std::vector<int32_t> want;
  int base = 0, rc;
  for (int i = 0; i < n; ++i) {
    const int at = hy.len[(size_t)e[i].seq];
    if ((rc = hy_kv_ensure(m, e[i].seq, at + e[i].n_tokens)) != KH_OK) return rc;
    es.push_back({e[i].seq, e[i].n_tokens, at, e[i].tokens});
    for (int k = 0; k < e[i].n_want; ++k) want.push_back(base + e[i].want[k]);
    base += e[i].n_tokens;
  }
  if (!want.empty() && !h_logits) return KH_ERR_INVALID_ARG;
  bool single = n <= hy_decode_max(m) && !hy.probe && !dbg_off("KH_HY_DECODE");
  for (const HyEntry& x : es) single = single && x.n == 1;
  if (single) {  // the fused decode step computes every sequence's logits
    std::vector<float> lg(want.empty() ? 0 : (size_t)n * hy.c.vocab);
    if ((rc = hy_decode(m, es.data(), n, want.empty() ? nullptr : lg.data())) != KH_OK) return rc;
    for (size_t k = 0; k < want.size(); ++k)
      memcpy(h_logits + k * hy.c.vocab, lg.data() + (size_t)want[k] * hy.c.vocab, (size_t)hy.c.vocab * 4);
  } else if ((rc = hy_forward(m, es.data(), n, want.data(), (int)want.size(), want.empty() ? nullptr : h_logits)) != KH_OK) return rc;
  for (int i = 0; i < n; ++i) hy.len[(size_t)e[i].seq] += e[i].n_tokens;
  return KH_OK;
}
// .bin models: one sequence, token by token through predict
int forward_bin(kh_model* m, const kh_batch_entry* e, int n, float* h_logits) {
  for (int i = 0; i < n; ++i)
    for (int k = 0, w = 0; k < e[i].n_tokens; ++k) {
      int32_t next = -1;
      int rc = kh_model_predict(m, e[i].tokens[k], m->seq_len[0], 1, KH_EXEC_FUSED, &next);
      if (rc != KH_OK) return rc;
      ++m->seq_len[0];
      if (w < e[i].n_want && e[i].want[w] == k) {
        if (!h_logits) return KH_ERR_INVALID_ARG;
        if ((rc = kh_model_get_logits(m, h_logits)) != KH_OK) return rc;
        h_logits += m->cfg.vocab_size;
        ++w;
      }
    }
  return KH_OK;
}
}  // namespace

extern "C" int kh_model_forward(kh_model* m, const kh_batch_entry* entries, int32_t n, float* h_logits) {
  if (!m || !entries || n <= 0) return KH_ERR_INVALID_ARG;
  return kh_api_guard([&]() -> int {
    const int rc = forward_checks(m, m->hy ? m->hy->len : m->seq_len, entries, n);
    if (rc != KH_OK) return rc;
    return m->hy ? forward_layers(m, entries, n, h_logits) : forward_bin(m, entries, n, h_logits);
  });
}

extern "C" int kh_model_generate_batch(kh_model* m, int32_t n, const int32_t* const* h_prompts, const int32_t* n_prompt,
                                       const int32_t* max_new, const int32_t* h_stop, int32_t n_stop, int32_t* h_out,
                                       int32_t cap, int32_t* h_n_out) {
  if (!m || n <= 0 || !h_prompts || !n_prompt || !max_new || !h_out || cap <= 0 || !h_n_out || n_stop < 0 || (n_stop && !h_stop))
    return KH_ERR_INVALID_ARG;
  if (!m->hy) return KH_ERR_UNSUPPORTED;
  for (int i = 0; i < n; ++i)
    if (max_new[i] <= 0 || max_new[i] > cap || n_prompt[i] <= 0) return KH_ERR_INVALID_ARG;
  return kh_api_guard([&]() -> int {
    std::vector<int32_t> seq((size_t)n, -1), last((size_t)n), at((size_t)n);
    int rc = KH_OK;
    for (int i = 0; i < n && rc == KH_OK; ++i) rc = kh_seq_open(m, &seq[(size_t)i]);
    const size_t V = (size_t)m->cfg.vocab_size;
    std::vector<float> lg(V * (size_t)n);
    std::vector<int> live;
    for (int i = 0; i < n; ++i) {
      live.push_back(i);
      h_n_out[i] = 0;
    }
    bool first = true;
    const int32_t zero = 0;
    while (rc == KH_OK && !live.empty()) {
      std::vector<kh_batch_entry> es;
      for (int i : live) {
        at[(size_t)i] = n_prompt[i] - 1;
        if (first) es.push_back({seq[(size_t)i], n_prompt[i], h_prompts[i], 1, &at[(size_t)i]});
        else es.push_back({seq[(size_t)i], 1, &last[(size_t)i], 1, &zero});
      }
      rc = kh_model_forward(m, es.data(), (int32_t)es.size(), lg.data());
      if (rc != KH_OK) break;
      first = false;
      std::vector<int> next;
      for (size_t k = 0; k < live.size(); ++k) {
        const int i = live[k];
        const float* z = lg.data() + k * V;
        const int32_t t = (int32_t)(std::max_element(z, z + V) - z);  // first maximum, like the sampler
        last[(size_t)i] = t;
        const bool stop = std::find(h_stop, h_stop + n_stop, t) != h_stop + n_stop;
        if (!stop) h_out[(size_t)i * cap + h_n_out[i]++] = t;
        if (stop || h_n_out[i] >= max_new[i]) {
          (void)kh_seq_close(m, seq[(size_t)i]);
          seq[(size_t)i] = -1;
        } else {
          next.push_back(i);
        }
      }
      live.swap(next);
    }
    for (int32_t q : seq)
      if (q >= 0) (void)kh_seq_close(m, q);
    return rc;
  });
}

extern "C" int kh_model_probe_residual(kh_model* m, float* h_buf, int64_t cap, int64_t* n_written) {
  if (!m || (h_buf && cap <= 0)) return KH_ERR_INVALID_ARG;
  if (!m->hy) return KH_ERR_UNSUPPORTED;
  if (n_written) *n_written = m->hy->probe_n;
  m->hy->probe = h_buf;
  m->hy->probe_cap = h_buf ? cap : 0;
  m->hy->probe_n = 0;
  return KH_OK;
}
