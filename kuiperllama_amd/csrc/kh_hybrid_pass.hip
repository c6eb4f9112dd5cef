// kh_hybrid_pass.hip — layer-list models: one pass over T tokens of any number of sequences.  The tokens of all
// entries are concatenated (no padding); linear layers see one [T, K] matrix, the mixers find each token's sequence
// through the pass tables, and every sequence continues from the cache rows and the recurrent state of its slot.
#include <stdio.h>
#include <string.h>

#include <algorithm>

#include "kh_expanded.h"
#include "kh_hybrid.h"

using namespace khm;

namespace {

#define TRY(e)                       \
  do {                               \
    const int _rc = (e);             \
    if (_rc != KH_OK) return _rc;    \
  } while (0)

// Query-row tiles of an attention kernel: `per` rows a token, `lanes` workgroups per tile (key / value heads), big tiles of
// `big` rows.  Layers of one kind share a tile list.
struct RowKind {
  int per, lanes, big;
  bool operator==(const RowKind& o) const { return per == o.per && lanes == o.lanes && big == o.big; }
};
struct RowTiles {
  RowKind kind;
  int rows, off, n;  // rows of a tile; offset in ints from the table base; tiles
};
struct PassSeg {
  int slot, row0, n, pos0;
};
// device view of one pass
struct Pass {
  std::vector<PassSeg> segs;
  bool expand = false;  // few long segments: latent attention in its expanded form
  int T = 0, S = 0, n_chunks = 0, n_multi_segs = 0, n_multi_chunks = 0, n_want = 0;
  PassTabs p{};
  const ScanChunk* chunks = nullptr;
  const int32_t *multi0 = nullptr, *multin = nullptr, *want = nullptr;
  const int32_t* base = nullptr;
  std::vector<RowTiles> tiles;
  bool no_logits = false;  // nothing of the last layer's output is wanted: only its cache rows / state
};

// ---- tables ------------------------------------------------------------------------------------------------------
struct TabBuilder {
  std::vector<int32_t> v;
  int put(const int32_t* p, size_t n) {
    const size_t o = (v.size() + 3) / 4 * 4;
    v.resize(o + n);
    if (n) memcpy(v.data() + o, p, n * 4);
    return (int)o;
  }
  int put(const std::vector<int32_t>& x) { return put(x.data(), x.size()); }
};

// latents of more than 256: 32 rows, the accumulators of 64 would not fit
RowKind row_kind(const HyLatent& la) { return {la.H, 1, la.Rp > 256 ? 32 : 64}; }
RowKind row_kind(const Hybrid& hy, const HyHeads& a) { return {a.H / a.G, a.G, heads_wide_rows(a.dkp, a.dvp, hy.elem()) ? 128 : 64}; }
std::vector<RowKind> row_kinds(const Hybrid& hy) {
  std::vector<RowKind> r;
  for (auto& l : hy.layers) {
    if (l.mixer == HY_MAMBA1) continue;
    const RowKind k = l.mixer == HY_LATENT ? row_kind(l.la) : row_kind(hy, l.ha);
    if (std::find(r.begin(), r.end(), k) == r.end()) r.push_back(k);
  }
  return r;
}
// big tiles, or 64 rows where 128 would not give every CU two workgroups, or 16 where the rows of the segments would
// leave most of those empty
int row_tiles(const std::vector<int32_t>& seg_n, const RowKind& kind, std::vector<int32_t>* tab) {
  long rows = 0, t64 = 0, big = 0;
  for (int n : seg_n) {
    rows += (long)n * kind.per;
    t64 += ((long)n * kind.per + 63) / 64;
    big += ((long)n * kind.per + kind.big - 1) / kind.big;
  }
  int step = t64 * 64 > 2 * rows ? 16 : (kind.big > 64 && big * kind.lanes < 512 ? 64 : kind.big);
  if (const char* e = dbg("KH_HY_ROWS")) step = atoi(e) == 16 ? 16 : std::min(atoi(e) == 128 ? 128 : 64, kind.big);
  tab->clear();
  for (size_t s = 0; s < seg_n.size(); ++s)
    for (int r = (seg_n[s] * kind.per - 1) / step * step; r >= 0; r -= step) {  // the longest key ranges first
      tab->push_back((int)s);
      tab->push_back(r);
    }
  return step;
}

// ---- the pass ----------------------------------------------------------------------------------------------------
template <class T>
struct Runner {
  kh_model* m;
  Hybrid& hy;
  const Pass& ps;
  hipStream_t s;
  AddArgs<T> pend{};
  const T* pend_xn2 = nullptr;

  Runner(kh_model* mm, const Pass& p) : m(mm), hy(*mm->hy), ps(p), s(mm->stream) {}

  LgArgs gemm(const HyMat& w, const void* X, int ldx, void* out, int ldo) {
    LgArgs a{};
    a.W = w.w;
    a.X = X;
    a.out = out;
    a.M = ps.T;
    a.N = w.N;
    a.K = w.ld;
    a.ldw = w.ld;
    a.ldx = ldx;
    a.ldo = ldo;
    return a;
  }
  // x += everything pending (+ the loop entry); layer != nullptr: its norms
  int combine(const HyLayer* l, bool from_embed, int pass_no, T* cat = nullptr) {
    CombineArgs<T> a{};
    a.x = hy.x;
    a.x0 = hy.x0;
    a.add = pend;
    a.embed = (const T*)hy.embed.w;
    a.pos_emb = (const T*)hy.pos_emb.w;
    a.tok = ps.p.tok;
    a.pos = ps.p.pos;
    a.cat = cat;
    a.W = hy.c.width;
    a.ld = hy.c.widthp;
    a.from_embed = from_embed;
    a.add_x0 = pass_no > 0 && !hy.enter.N;
    a.step = pass_no >= 0 && hy.step.on ? hy.step.p + (size_t)pass_no * hy.c.widthp : nullptr;
    a.rms = hy.c.rms;
    a.eps = hy.c.eps;
    a.mult = hy.c.mult;
    a.emb_scale = hy.c.emb_scale;
    a.xn2_prev = (const T*)hy.xn2;
    a.xn1 = (T*)hy.xn1;
    a.xn2 = (T*)hy.xn2;
    if (l) {
      a.w1 = l->n1.p;
      a.b1 = l->n1b.p;
      if (l->ff.on && l->n2.on) {
        a.w2 = l->n2.p;
        a.b2 = l->n2b.p;
      }
    }
    pend = AddArgs<T>{};
    hipLaunchKernelGGL(k_combine<T>, dim3(ps.T), dim3(256), (size_t)hy.c.widthp * 4, s, a);
    return KH_OK;
  }

  // a pass of the loop starts: x <- W [x ; embedding output]
  int enter(bool from_embed) {
    const int Wp = hy.c.widthp;
    TRY(combine(nullptr, from_embed, -1, (T*)hy.a2));
    return lg_launch<T, LG_F32>(s, gemm(hy.enter, hy.a2, 2 * Wp, hy.x, Wp));
  }

  int heads(const HyRun& r, const HyHeads& ha, bool state_only) {
    LgArgs pr = gemm(ha.qkvg, hy.xn1, hy.c.widthp, hy.a1, ha.qkvg.N);
    pr.bias = ha.qkvg_b.p;
    if (state_only) {  // key and value rows only
      pr.W = (const T*)ha.qkvg.w + (size_t)ha.k_off() * ha.qkvg.ld;
      pr.out = (T*)hy.a1 + ha.k_off();
      pr.N = ha.g_off() - ha.k_off();
      if (pr.bias) pr.bias += ha.k_off();
    }
    TRY((lg_launch<T, LG_T>(s, pr)));
    HeadRowsArgs<T> hr{ha.head_row(hy.c.eps), (const T*)hy.a1, (T*)m->kcache + r.kv_off, hy.kv_slot, ha.qkvg.N, ps.T, ps.p};
    hipLaunchKernelGGL(k_heads_rows<T>, dim3((ps.T * ha.G + 3) / 4), dim3(256), 0, s, hr);
    if (state_only) return KH_OK;
    const RowTiles* rt = row_tiles_of(row_kind(hy, ha));
    if (!rt) return KH_ERR_INTERNAL;
    HeadsArgs a = heads_args(hy, ha, (const T*)m->kcache + r.kv_off);
    a.raw = hy.a1;
    a.ldr = ha.qkvg.N;
    a.out = hy.a0;
    a.ldo = ha.o.ld;
    a.nsplit = 1;
    a.tiles = (const LatTile*)(ps.base + rt->off);
    a.p = ps.p;
    TRY(heads_attn_launch<T>(s, a, rt->n, rt->rows));
    LgArgs o = gemm(ha.o, hy.a0, ha.o.ld, hy.mix, hy.c.widthp);
    o.bias = ha.o_b.p;
    return lg_launch<T, LG_F32>(s, o);
  }
  const RowTiles* row_tiles_of(const RowKind& k) const {
    for (auto& t : ps.tiles)
      if (t.kind == k) return &t;
    return nullptr;
  }

  int mamba(const HyRun& r, const HyMamba& mb, bool state_only) {
    const int I = mb.inner, N = mb.state;
    TRY((lg_launch<T, LG_T>(s, gemm(mb.in, hy.xn1, hy.c.widthp, hy.a0, 2 * I))));
    ConvArgs<T> cv{};
    cv.xz = (const T*)hy.a0;
    cv.out = (T*)hy.a1;
    cv.w = mb.conv.p;
    cv.b = mb.conv_b.p;
    cv.state = hy.state + r.conv_off;
    cv.slot_stride = hy.st_slot;
    cv.C = I;
    cv.ldx = 2 * I;
    cv.ldo = mb.innerp;
    cv.taps = mb.taps;
    cv.p = ps.p;
    conv_launch<T>(s, cv, ps.T);
    hipLaunchKernelGGL(k_conv_state<T>, dim3((I + 255) / 256, ps.S), dim3(256), 0, s, cv);
    {
      LgArgs a = gemm(mb.x, hy.a1, mb.innerp, hy.a2, mb.rankp);
      a.n_split = mb.rankp;
      a.out2 = hy.bc;
      a.ldo2 = 2 * N;
      TRY((lg_launch<T, LG_SPLIT>(s, a)));
    }
    {
      LgArgs a = gemm(mb.dt, hy.a2, mb.rankp, hy.dt, I);
      a.bias = mb.dt_b.p;
      TRY((lg_launch<T, LG_SOFTPLUS>(s, a)));
    }
    ScanArgs<T> sc{};
    sc.x = (const T*)hy.a1;
    sc.z = (const T*)hy.a0 + I;
    sc.dt = hy.dt;
    sc.bc = hy.bc;
    sc.A2 = mb.A2.p;
    sc.D = mb.D.p;
    sc.out = (T*)hy.a2;
    sc.state = hy.state + r.st_off;
    sc.slot_stride = hy.st_slot;
    sc.ends = hy.ends;
    sc.dtsum = hy.dtsum;
    sc.chunks = ps.chunks;
    sc.p = ps.p;
    sc.C = I;
    sc.N = N;
    sc.ldx = mb.innerp;
    sc.ldz = 2 * I;
    sc.ldo = mb.innerp;
    if (ps.n_multi_segs) {
      TRY((scan_launch<T, false>(s, sc, ps.n_multi_chunks)));
      hipLaunchKernelGGL(k_scan_carry<T>, dim3((unsigned)(((size_t)I * N + 255) / 256), ps.n_multi_segs), dim3(256), 0, s, sc,
                         ps.multi0, ps.multin);
    }
    TRY((scan_launch<T, true>(s, sc, ps.n_chunks)));
    if (state_only) return KH_OK;
    return lg_launch<T, LG_F32>(s, gemm(mb.o, hy.a2, mb.innerp, hy.mix, hy.c.widthp));
  }

  // keys and values of every head of one segment, rebuilt from its cached latents, and its attention: q in a1 -> a0
  int expanded(const HyRun& r, const HyLatent& la, const PassSeg& sg) {
    const int H = la.H, keys = sg.pos0 + sg.n;
    const T* cache = (const T*)m->kcache + (size_t)sg.slot * hy.kv_slot + r.kv_off;
    LgArgs k = gemm(la.uk, cache, la.row(), hy.kx, H * la.dnp);
    k.M = keys;
    TRY((lg_launch<T, LG_T>(s, k)));
    LgArgs v{};  // transposed: features are the keys
    v.W = cache;
    v.X = la.uv.w;
    v.out = hy.vx;
    v.M = H * la.dvp;
    v.N = keys;
    v.K = la.Rp;
    v.ldw = la.row();
    v.ldx = la.Rp;
    v.ldo = hy.exp_keys;
    TRY((lg_launch<T, LG_T>(s, v)));
    ExpArgs a{hy.a1, hy.kx, hy.vx, cache + la.Rp, la.sink.p, hy.a0, H, la.dnp, la.drp, la.dvp, la.row(), hy.exp_keys,
              sg.row0, sg.n, sg.pos0, la.scale * 1.44269504088896f};
    return exp_attn_launch<T>(s, a);
  }

  int latent(const HyRun& r, const HyLatent& la, bool state_only) {
    const int H = la.H, row = la.row(), qh = la.dnp + la.drp;
    TRY((lg_launch<T, LG_F32>(s, gemm(la.dqkv, hy.xn1, hy.c.widthp, hy.f32a, la.dqkv.N))));
    LatPrepArgs<T> lp{};
    lp.raw = hy.f32a;
    lp.qn = la.qn.p;
    lp.kvn = la.kvn.p;
    lp.rope = la.rope;
    lp.cq = (T*)hy.a0;
    lp.cache = (T*)m->kcache + r.kv_off;
    lp.slot_elems = hy.kv_slot;
    lp.ldr = la.dqkv.N;
    lp.ldq = la.qrp;
    lp.qr = la.qr;
    lp.R = la.R;
    lp.dr = la.dr;
    lp.Rp = la.Rp;
    lp.row = row;
    lp.dims = la.dims;
    lp.eps = hy.c.eps;
    lp.p = ps.p;
    hipLaunchKernelGGL(k_latent_prep<T>, dim3(ps.T), dim3(256), 0, s, lp);
    if (state_only) return KH_OK;
    TRY((lg_launch<T, LG_T>(s, gemm(la.uq, hy.a0, la.qrp, hy.a1, H * qh))));
    if (ps.expand && la.scale > 0.f && exp_supported(la.dnp, la.drp, la.dvp)) {
      if (la.dims)
        hipLaunchKernelGGL(k_rope_inplace<T>, dim3(ps.T), dim3(256), 0, s, (T*)hy.a1, la.rope, H, la.dnp, la.drp, la.dims, ps.p);
      for (const PassSeg& sg : ps.segs) TRY(expanded(r, la, sg));
      return lg_launch<T, LG_F32>(s, gemm(la.o, hy.a0, H * la.dvp, hy.mix, hy.c.widthp));
    }
    {  // absorbed queries: per head, W_uk^T q_n
      LgArgs a = gemm(la.ukT, hy.a1, H * qh, hy.a2, H * row);
      a.N = la.Rp;
      a.w_z = (size_t)la.Rp * la.dnp;
      a.x_z = (size_t)qh;
      a.o_z = (size_t)row;
      TRY((lg_launch<T, LG_T>(s, a, H)));
    }
    RopeQArgs<T> rq{(const T*)hy.a1, (T*)hy.a2, la.rope, H, la.dnp, la.dr, la.drp, la.Rp, la.dims, ps.p};
    if (la.drp) hipLaunchKernelGGL(k_rope_q<T>, dim3(ps.T), dim3(256), 0, s, rq);
    const RowTiles* lt = row_tiles_of(row_kind(la));
    if (!lt) return KH_ERR_INTERNAL;
    LatArgs at{};
    at.Q = hy.a2;
    at.cache = (const T*)m->kcache + r.kv_off;
    at.slot_elems = hy.kv_slot;
    at.sink = la.sink.p;
    at.out = hy.a0;
    at.tiles = (const LatTile*)(ps.base + lt->off);
    at.H = H;
    at.Rp = la.Rp;
    at.row = row;
    at.nsplit = 1;
    at.scale2 = la.scale * 1.44269504088896f;
    at.p = ps.p;
    TRY(lat_attn_launch<T>(s, at, lt->n, 64 / lt->rows));
    {  // values: per head, W_uv o
      LgArgs a = gemm(la.uv, hy.a0, H * la.Rp, hy.a1, H * la.dvp);
      a.N = la.dvp;
      a.w_z = (size_t)la.dvp * la.Rp;
      a.x_z = (size_t)la.Rp;
      a.o_z = (size_t)la.dvp;
      TRY((lg_launch<T, LG_T>(s, a, H)));
    }
    return lg_launch<T, LG_F32>(s, gemm(la.o, hy.a1, H * la.dvp, hy.mix, hy.c.widthp));
  }

  int feed_forward(const HyMoe& f, const void* in) {
    if (f.top) TRY(experts(f, in));
    if (f.sff) {
      const int Wp = hy.c.widthp;
      LgArgs a = gemm(f.sgu, in, Wp, hy.hs, f.sffp);
      a.act = f.sact;
      TRY((lg_launch<T, LG_GATED>(s, a)));
      TRY((lg_launch<T, LG_T>(s, gemm(f.sdown, hy.hs, f.sffp, hy.sh, Wp))));
      pend.sh = (const T*)hy.sh;
      pend.sh_g = f.sgate ? hy.sh_g : nullptr;
    }
    return KH_OK;
  }
  int experts(const HyMoe& f, const void* in) {
    const int W = hy.c.width, Wp = hy.c.widthp;
    TRY((lg_launch<T, LG_F32>(s, gemm(f.zr, in, Wp, hy.z, f.zr.N))));
    RouteArgs ra{hy.z, f.corr.p, hy.moe_id, hy.moe_w, hy.id_w, hy.sh_g, ps.T, f.zr.N, f.n_out(), f.E, f.top, f.sgate, f.over_chosen};
    moe_route_launch(s, ra);
    const int bm = lg_group_bm((long)ps.T * f.top, f.n_out());
    ListArgs li{hy.moe_id, hy.moe_rows, hy.moe_slot, hy.tiles, hy.n_tiles, ps.T, f.top, f.E, bm};
    hipLaunchKernelGGL(k_moe_lists, dim3(1), dim3(1024), 0, s, li);
    const long rows = (long)ps.T * f.top;
    const int mt = (int)(rows / bm + std::min<long>(f.E, rows));
    {
      LgArgs a = gemm(f.gu, in, Wp, hy.h, f.ffp);
      a.N = 2 * f.ffp;
      a.act = f.act;
      a.tiles = hy.tiles;
      a.n_tiles = hy.n_tiles;
      a.gather = hy.moe_rows;
      a.w_group = (size_t)2 * f.ffp * f.gu.ld;
      TRY((lg_launch<T, LG_GATED>(s, a, 1, bm, mt)));
    }
    {
      LgArgs a = gemm(f.down, hy.h, f.ffp, hy.y, Wp);
      a.N = W;
      a.tiles = hy.tiles;
      a.n_tiles = hy.n_tiles;
      a.w_group = (size_t)W * f.down.ld;
      TRY((lg_launch<T, LG_T>(s, a, 1, bm, mt)));
    }
    pend.y = (const T*)hy.y;
    pend.y_slot = hy.moe_slot;
    pend.y_w = hy.moe_w;
    pend.id_w = f.ident ? hy.id_w : nullptr;
    pend.top = f.top;
    return KH_OK;
  }

  int layers() {
    for (size_t i = 0; i < hy.runs.size(); ++i) {
      const HyRun& r = hy.runs[i];
      const HyLayer& l = hy.layers[(size_t)r.layer];
      const bool state_only = ps.no_logits && i + 1 == hy.runs.size() && !hy.probe;
      const bool through = r.pass >= 0 && hy.enter.N;
      if (through) TRY(enter(i == 0));
      TRY(combine(&l, i == 0 && !through, r.pass));
      TRY(l.mixer == HY_MAMBA1 ? mamba(r, l.mb, state_only)
          : l.mixer == HY_LATENT ? latent(r, l.la, state_only) : heads(r, l.ha, state_only));
      if (state_only) break;
      pend.mix = hy.mix;
      if (l.ff.on) TRY(feed_forward(l.ff, l.n2.on ? hy.xn2 : hy.xn1));
      if (hy.probe) {
        TRY(combine(nullptr, false, -1));
        const int64_t n = (int64_t)ps.T * hy.c.width;
        if (hy.probe_n + n <= hy.probe_cap) {
          KH_CHECK_HIP(hipMemcpy2DAsync(hy.probe + hy.probe_n, (size_t)hy.c.width * 4, hy.x, (size_t)hy.c.widthp * 4,
                                        (size_t)hy.c.width * 4, (size_t)ps.T, hipMemcpyDeviceToHost, s));
          KH_CHECK_HIP(hipStreamSynchronize(s));
          hy.probe_n += n;
        }
      }
    }
    return kh_launch_status();
  }
  // logits of rows[0 .. n) (device list) -> out [n][vocab]; n <= wl_rows
  int logits(const int32_t* rows, int n, float* out) {
    hipLaunchKernelGGL(k_gather_norm<T>, dim3(n), dim3(256), 0, s, (const float*)hy.x, rows, hy.fnorm.p, hy.fnorm_b.p,
                       (T*)hy.xw, hy.c.width, hy.c.widthp, hy.c.eps, (int)hy.c.rms);
    LgArgs a = gemm(hy.head, hy.xw, hy.c.widthp, out, hy.c.vocab);
    a.M = n;
    a.cap = hy.c.cap;
    TRY((lg_launch<T, LG_SOFTCAP>(s, a)));
    return kh_launch_status();
  }
};

template <class T>
int run_pass(kh_model* m, const Pass& ps, float* h_logits) {
  Hybrid& hy = *m->hy;
  Runner<T> r(m, ps);
  TRY(r.layers());
  if (!ps.n_want) return KH_OK;
  TRY(r.combine(nullptr, false, -1));
  for (int w = 0; w < ps.n_want; w += hy.wl_rows) {
    const int n = std::min(hy.wl_rows, ps.n_want - w);
    TRY(r.logits(ps.want + w, n, hy.wlogits));
    KH_CHECK_HIP(hipMemcpyAsync(h_logits + (size_t)w * hy.c.vocab, hy.wlogits, (size_t)n * hy.c.vocab * 4,
                                hipMemcpyDeviceToHost, m->stream));
  }
  return KH_OK;
}

}  // namespace

namespace khm {

static __global__ void k_one_partial(const int32_t* idx, float* val, int32_t* out, int n) {
  for (int i = threadIdx.x; i < n; i += 64) {
    val[i] = i ? -INFINITY : 0.f;
    out[i] = *idx;
  }
}
int hy_argmax_partial(kh_model* m) {
  TRY(kh_argmax_f32(m->logits, m->cfg.vocab_size, m->d_next, (void*)m->stream));
  hipLaunchKernelGGL(k_one_partial, dim3(1), dim3(64), 0, m->stream, (const int32_t*)m->d_next, m->part_val, m->part_idx, m->nparts);
  return kh_launch_status();
}

int hy_forward(kh_model* m, const HyEntry* e, int n, const int32_t* want, int n_want, float* h_logits) {
  Hybrid& hy = *m->hy;
  KH_CHECK_HIP(hipSetDevice(m->opts.device));
  KH_CHECK_HIP(hipStreamSynchronize(m->stream));  // the pinned tables of the call before are free again
  const std::vector<RowKind> kinds = row_kinds(hy);
  // ---- cut the concatenated tokens into passes and build every pass's tables
  std::vector<Pass> passes;
  std::vector<int32_t> all;
  struct Off {
    int tok, pos, seg, slot, row0, sn, pos0, ck, m0, mn, want;
  };
  std::vector<Off> offs;
  std::vector<size_t> bases;
  int ei = 0, eo = 0, row_base = 0, wi = 0, exp_keys = 0;
  while (ei < n) {
    std::vector<int32_t> tok, pos, seg, slot, row0, sn, pos0, single, multi, m0, mn, wr, lt;
    while (ei < n && (int)tok.size() < hy.tmax) {
      const HyEntry& x = e[ei];
      const int k = std::min(x.n - eo, hy.tmax - (int)tok.size());
      const int sg = (int)slot.size();
      slot.push_back(x.slot);
      row0.push_back((int)tok.size());
      sn.push_back(k);
      pos0.push_back(x.pos0 + eo);
      const int nck = (k + KH_SCAN_CH - 1) / KH_SCAN_CH;
      std::vector<int32_t>& dst = nck > 1 ? multi : single;
      if (nck > 1) {
        m0.push_back((int)multi.size() / 4);
        mn.push_back(nck);
      }
      for (int c = 0; c < nck; ++c) {
        const int r = c * KH_SCAN_CH;
        for (int v : {sg, (int)tok.size() + r, std::min(KH_SCAN_CH, k - r), (c == 0 ? 1 : 0) | (c + 1 == nck ? 2 : 0)})
          dst.push_back(v);
      }
      for (int i = 0; i < k; ++i) {
        tok.push_back(x.tok[eo + i]);
        pos.push_back(x.pos0 + eo + i);
        seg.push_back(sg);
      }
      eo += k;
      if (eo == x.n) {
        ++ei;
        eo = 0;
      }
    }
    Pass p;
    p.T = (int)tok.size();
    p.S = (int)slot.size();
    p.n_multi_chunks = (int)multi.size() / 4;
    p.n_multi_segs = (int)m0.size();
    p.n_chunks = p.n_multi_chunks + (int)single.size() / 4;
    while (wi < n_want && want[wi] < row_base + p.T) wr.push_back(want[wi++] - row_base);
    p.n_want = (int)wr.size();
    p.no_logits = wr.empty();
    p.expand = hy.any_latent && p.S <= 8 && !dbg_off("KH_HY_EXPAND");
    for (int i = 0; i < p.S; ++i) {
      p.segs.push_back({slot[(size_t)i], row0[(size_t)i], sn[(size_t)i], pos0[(size_t)i]});
      p.expand = p.expand && sn[(size_t)i] >= 32;
    }
    if (p.expand)
      for (const PassSeg& sg : p.segs) exp_keys = std::max(exp_keys, sg.pos0 + sg.n);
    row_base += p.T;
    multi.insert(multi.end(), single.begin(), single.end());
    TabBuilder tb;
    Off o;
    o.tok = tb.put(tok);
    o.pos = tb.put(pos);
    o.seg = tb.put(seg);
    o.slot = tb.put(slot);
    o.row0 = tb.put(row0);
    o.sn = tb.put(sn);
    o.pos0 = tb.put(pos0);
    o.ck = tb.put(multi);
    o.m0 = tb.put(m0);
    o.mn = tb.put(mn);
    o.want = tb.put(wr);
    for (const RowKind& kd : kinds) {
      RowTiles t{kd, row_tiles(sn, kd, &lt), 0, (int)lt.size() / 2};
      t.off = tb.put(lt);
      p.tiles.push_back(t);
    }
    bases.push_back((all.size() + 15) / 16 * 16);
    all.resize(bases.back() + tb.v.size());
    memcpy(all.data() + bases.back(), tb.v.data(), tb.v.size() * 4);
    offs.push_back(o);
    passes.push_back(std::move(p));
  }
  if (exp_keys > hy.exp_keys) TRY(hy_expand_buffers(m, exp_keys));
  // ---- upload
  if (all.size() > hy.tab_cap) {
    if (hy.h_tab) (void)hipHostFree(hy.h_tab);
    if (hy.d_tab) (void)hipFree(hy.d_tab);
    hy.h_tab = hy.d_tab = nullptr;
    hy.tab_cap = 0;
    const size_t cap = std::max<size_t>(all.size() * 2, 1 << 15);
    KH_CHECK_HIP(hipHostMalloc((void**)&hy.h_tab, cap * 4, hipHostMallocDefault));
    TRY(dalloc(&hy.d_tab, cap));
    hy.tab_cap = cap;
  }
  memcpy(hy.h_tab, all.data(), all.size() * 4);
  KH_CHECK_HIP(hipMemcpyAsync(hy.d_tab, hy.h_tab, all.size() * 4, hipMemcpyHostToDevice, m->stream));
  float* out = h_logits;
  for (size_t i = 0; i < passes.size(); ++i) {
    Pass& p = passes[i];
    const Off& o = offs[i];
    const int32_t* b = hy.d_tab + bases[i];
    p.base = b;
    p.p = PassTabs{b + o.tok, b + o.pos, b + o.seg, b + o.slot, b + o.row0, b + o.sn, b + o.pos0};
    p.chunks = (const ScanChunk*)(b + o.ck);
    p.multi0 = b + o.m0;
    p.multin = b + o.mn;
    p.want = b + o.want;
    TRY(hy.f32 ? run_pass<float>(m, p, out) : run_pass<bf16>(m, p, out));
    if (out) out += (size_t)p.n_want * hy.c.vocab;
  }
  if (h_logits) KH_CHECK_HIP(hipStreamSynchronize(m->stream));
  return KH_OK;
}

// ---- one token, everything on the device -------------------------------------------------------------------------
static __global__ void k_one_tabs(const int32_t* d_token, const int32_t* d_pos, int32_t* tab) {
  if (threadIdx.x == 0) {
    tab[0] = *d_token;
    tab[1] = tab[6] = *d_pos;  // position of the token, and of the segment's first row
  }
}
// tab: tok, pos, seg, slot, row0, n, pos0, (pad), chunk[4], want, (pad) 3, tiles ...
int hy_unfused_step(kh_model* m) {
  Hybrid& hy = *m->hy;
  Pass p;
  std::vector<int32_t> tab{0, 0, 0, 0, 0, 1, 0, 0, 0, 0, 1, 3, 0, 0, 0, 0}, lt;
  for (const RowKind& kd : row_kinds(hy)) {
    const int rows = row_tiles({1}, kd, &lt);
    p.tiles.push_back({kd, rows, (int)tab.size(), (int)lt.size() / 2});
    tab.insert(tab.end(), lt.begin(), lt.end());
  }
  if (!hy.d_one) {
    TRY(dalloc(&hy.d_one, tab.size()));
    KH_CHECK_HIP(hipMemcpyAsync(hy.d_one, tab.data(), tab.size() * 4, hipMemcpyHostToDevice, m->stream));
    KH_CHECK_HIP(hipStreamSynchronize(m->stream));
  }
  hipLaunchKernelGGL(k_one_tabs, dim3(1), dim3(64), 0, m->stream, (const int32_t*)m->d_token, (const int32_t*)m->d_pos, hy.d_one);
  const int32_t* b = hy.d_one;
  p.T = p.S = p.n_chunks = 1;
  p.base = b;
  p.p = PassTabs{b, b + 1, b + 2, b + 3, b + 4, b + 5, b + 6};
  p.chunks = (const ScanChunk*)(b + 8);
  p.want = b + 12;
  auto go = [&](auto r) -> int {
    TRY(r.layers());
    TRY(r.combine(nullptr, false, -1));
    return r.logits(p.want, 1, m->logits);
  };
  return hy.f32 ? go(Runner<float>(m, p)) : go(Runner<bf16>(m, p));
}
}  // namespace khm
