// kh_hybrid_load.hip — layer-list models: registry, config.json, model.safetensors -> padded weight rows in one HBM
// arena, and the state manager (recurrent state, latent and key / value cache of every sequence slot).
//
// Weight rows are re-laid once at load for the kernels that read them: row lengths padded to KH_LPAD elements with
// zeros, matrices that share an input stacked (router + shared gate; query and key/value down-projections; query, key,
// value and gate heads), gate and up rows interleaved in groups of 16, W_uk transposed per head, latent heads padded to
// KH_LPAD, plain heads to 16 rows.  A learned distance bias becomes a table by distance.
#include <fcntl.h>
#include <math.h>
#include <stdio.h>
#include <string.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <algorithm>
#include <atomic>
#include <map>
#include <thread>

#include "kh_hybrid.h"

using namespace khm;

namespace {

int pad_to(int v, int g) { return (v + g - 1) / g * g; }
int padk(int v) { return pad_to(v, KH_LPAD); }

float bf16_to_f(uint16_t u) {
  const uint32_t w = (uint32_t)u << 16;
  float f;
  memcpy(&f, &w, 4);
  return f;
}
uint16_t f_to_bf16(float f) {  // round to nearest even
  uint32_t u;
  memcpy(&u, &f, 4);
  if ((u & 0x7fffffffu) > 0x7f800000u) return (uint16_t)((u >> 16) | 0x40);
  return (uint16_t)((u + 0x7fffu + ((u >> 16) & 1u)) >> 16);
}

// ---- safetensors: 8-byte little-endian header length, JSON name -> dtype, shape, data_offsets, data -------------
struct Tensor {
  const char* p = nullptr;
  int kind = 0;  // 0 bf16, 1 fp32, 2 fp16 (not accepted), 3 int32
  std::vector<int64_t> shape;
  int64_t n() const {
    int64_t k = 1;
    for (int64_t s : shape) k *= s;
    return k;
  }
  float at(int64_t i) const {
    if (kind == 1) {
      float f;
      memcpy(&f, p + 4 * i, 4);
      return f;
    }
    uint16_t u;
    memcpy(&u, p + 2 * i, 2);
    return bf16_to_f(u);
  }
};
struct Tensors {
  std::map<std::string, Tensor> t;
  std::string missing;  // first name that was asked for in vain or had an unexpected shape
  int parse(const char* data, size_t nbytes) {
    if (nbytes < 8) return KH_ERR_FORMAT;
    uint64_t hl = 0;
    for (int i = 7; i >= 0; --i) hl = hl << 8 | (unsigned char)data[i];
    if (hl > nbytes - 8) return KH_ERR_FORMAT;
    Json j{data + 8, data + 8 + hl};
    JsonValue v;
    if (!json_parse(j, &v) || v.kind != JsonValue::OBJ) return KH_ERR_FORMAT;
    const char* base = data + 8 + hl;
    const uint64_t room = nbytes - 8 - hl;
    for (auto& kv : v.obj) {
      if (kv.first == "__metadata__") continue;
      Tensor x;
      const std::string d = kv.second.text("dtype");
      int es = 2;
      if (d == "BF16") x.kind = 0;
      else if (d == "F32") x.kind = 1, es = 4;
      else if (d == "I32") x.kind = 3, es = 4;
      else return KH_ERR_UNSUPPORTED;
      const JsonValue *sh = kv.second.get("shape"), *of = kv.second.get("data_offsets");
      if (!sh || !of || of->arr.size() != 2) return KH_ERR_FORMAT;
      uint64_t n = 1;
      for (auto& s : sh->arr) {
        if (s.num < 0 || s.num > 2147483647.0) return KH_ERR_FORMAT;
        x.shape.push_back((int64_t)s.num);
        n *= (uint64_t)s.num;
      }
      const double o0 = of->arr[0].num, o1 = of->arr[1].num;
      if (o0 < 0 || o1 < o0 || o1 > (double)room || (uint64_t)(o1 - o0) != n * es) return KH_ERR_FORMAT;
      x.p = base + (uint64_t)o0;
      t[kv.first] = x;
    }
    return KH_OK;
  }
  bool has(const std::string& n) const { return t.count(n) != 0; }
  int64_t dim(const std::string& n, int i) const {
    auto it = t.find(n);
    return it == t.end() || i >= (int)it->second.shape.size() ? -1 : it->second.shape[(size_t)i];
  }
  // shape check; a mismatch is remembered in `missing`
  const Tensor* need(const std::string& n, std::vector<int64_t> shape) {
    auto it = t.find(n);
    if (it == t.end() || it->second.shape != shape || it->second.kind > 1) {
      if (missing.empty()) missing = n;
      return nullptr;
    }
    return &it->second;
  }
};

// ---- arena plan: what is copied where, executed by a team of threads ------------------------------------------
struct Plan {
  struct Job {  // rows [r0, r0 + n) of a source matrix -> destination rows, or its transpose
    const Tensor* t;
    int64_t src_row, rows, cols, src_col0, src_ld;  // source block
    size_t dst;                                     // element offset of destination row 0
    int ld;
    bool transpose;  // destination row = source column
  };
  std::vector<Job> jobs;
  size_t elems = 0, floats = 0;
  std::vector<std::pair<size_t, std::vector<float>>> vecs;
  size_t align(size_t v, size_t g) { return (v + g - 1) / g * g; }
  HyMat mat(int N, int K, int ld) {
    HyMat m;
    m.N = N;
    m.K = K;
    m.ld = ld;
    elems = align(elems, 512);
    m.off = elems;
    elems += (size_t)N * ld;
    return m;
  }
  // copy `rows` rows of t starting at src_row to rows dst_row.. of m, columns [c0, c0 + cols) to columns dst_col..
  void put(const HyMat& m, int64_t dst_row, const Tensor* t, int64_t src_row, int64_t rows, int64_t c0 = 0,
           int64_t cols = -1, int64_t dst_col = 0) {
    if (!t || rows <= 0) return;
    const int64_t ld = t->shape.size() > 1 ? t->shape[1] : t->shape[0];
    jobs.push_back({t, src_row, rows, cols < 0 ? ld : cols, c0, ld, m.off + (size_t)dst_row * m.ld + (size_t)dst_col,
                    m.ld, false});
  }
  void put_t(const HyMat& m, int64_t dst_row, const Tensor* t, int64_t src_row, int64_t rows) {
    if (!t || rows <= 0) return;
    jobs.push_back({t, src_row, rows, t->shape[1], 0, t->shape[1], m.off + (size_t)dst_row * m.ld, m.ld, true});
  }
  HyVec vec(std::vector<float> v) {
    HyVec r;
    floats = align(floats, 64);
    r.off = floats;
    r.on = true;
    floats += v.size();
    vecs.emplace_back(r.off, std::move(v));
    return r;
  }
  HyVec vec(const Tensor* t) {
    std::vector<float> v;
    if (t)
      for (int64_t i = 0; i < t->n(); ++i) v.push_back(t->at(i));
    return vec(std::move(v));
  }
  void run(bool f32, char* dst) const {
    std::atomic<size_t> next{0};
    auto work = [&] {
      for (size_t i; (i = next.fetch_add(1)) < jobs.size();) {
        const Job& j = jobs[i];
        for (int64_t r = 0; r < j.rows; ++r) {
          const int64_t s0 = (j.src_row + r) * j.src_ld + j.src_col0;
          if (!j.transpose && !f32 && j.t->kind == 0) {
            memcpy(dst + 2 * (j.dst + (size_t)r * j.ld), j.t->p + 2 * s0, 2 * (size_t)j.cols);
            continue;
          }
          for (int64_t c = 0; c < j.cols; ++c) {
            const size_t d = j.transpose ? j.dst + (size_t)c * j.ld + (size_t)r : j.dst + (size_t)r * j.ld + (size_t)c;
            const float v = j.t->at(s0 + c);
            if (f32) memcpy(dst + 4 * d, &v, 4);
            else {
              const uint16_t u = f_to_bf16(v);
              memcpy(dst + 2 * d, &u, 2);
            }
          }
        }
      }
    };
    const unsigned nt = std::max(1u, std::min(8u, std::thread::hardware_concurrency()));
    std::vector<std::thread> team;
    for (unsigned i = 1; i < nt; ++i) team.emplace_back(work);
    work();
    for (auto& t : team) t.join();
  }
};

// a vector of `heads` pieces of n elements, each padded with zeros to np
std::vector<float> head_vec(const Tensor* t, int heads, int n, int np) {
  std::vector<float> v((size_t)heads * np, 0.f);
  if (t)
    for (int h = 0; h < heads; ++h)
      for (int i = 0; i < n; ++i) v[(size_t)h * np + i] = t->at((int64_t)h * n + i);
  return v;
}

// gate and up rows interleaved in groups of 16: destination rows base + 32 (r / 16) + r % 16 (+ 16 for up)
void put_gate_up(Plan& pl, const HyMat& m, int64_t base, const Tensor* gate, const Tensor* up, int ff) {
  for (int r = 0; r < ff; r += 16) {
    const int n = ff - r < 16 ? ff - r : 16;
    pl.put(m, base + 2 * r, gate, r, n);
    pl.put(m, base + 2 * r + 16, up, r, n);
  }
}

// a size of the configuration, or the tensor shape's when the configuration leaves it out
int size_of(const JsonValue& v, const char* key, int64_t shape) {
  const JsonValue* x = v.get(key);
  if (x && x->kind == JsonValue::NUM) return (int)x->num;
  return shape > 0 && shape < (1 << 30) ? (int)shape : -1;
}

int load_mamba(Plan& pl, Tensors& ts, const std::string& p, const JsonValue& v, int W, HyMamba& mb) {
  mb.inner = size_of(v, "inner", ts.dim(p + ".A_log", 0));
  mb.state = size_of(v, "state", ts.dim(p + ".A_log", 1));
  mb.rank = size_of(v, "dt_rank", ts.dim(p + ".dt", 1));
  mb.taps = size_of(v, "conv", ts.dim(p + ".conv", 1));
  if (mb.inner <= 0 || mb.state <= 0 || mb.rank <= 0 || mb.taps <= 0) return KH_ERR_FORMAT;
  if (mb.taps > 64) return KH_ERR_UNSUPPORTED;
  if (mb.state > KH_SCAN_MAX_STATE) return KH_ERR_UNSUPPORTED;
  const int I = mb.inner, N = mb.state, r = mb.rank;
  mb.innerp = padk(I);
  mb.rankp = padk(r);
  mb.in = pl.mat(2 * I, W, padk(W));
  pl.put(mb.in, 0, ts.need(p + ".in", {2 * I, W}), 0, 2 * I);
  mb.x = pl.mat(mb.rankp + 2 * N, I, mb.innerp);
  const Tensor* x = ts.need(p + ".x", {r + 2 * N, I});
  pl.put(mb.x, 0, x, 0, r);
  pl.put(mb.x, mb.rankp, x, r, 2 * N);
  mb.dt = pl.mat(I, r, mb.rankp);
  pl.put(mb.dt, 0, ts.need(p + ".dt", {I, r}), 0, I);
  mb.o = pl.mat(W, I, mb.innerp);
  pl.put(mb.o, 0, ts.need(p + ".o", {W, I}), 0, W);
  mb.conv = pl.vec(ts.need(p + ".conv", {I, mb.taps}));
  mb.conv_b = pl.vec(ts.need(p + ".conv.b", {I}));
  mb.dt_b = pl.vec(ts.need(p + ".dt.b", {I}));
  std::vector<float> A2;
  if (const Tensor* a = ts.need(p + ".A_log", {I, N}))
    for (int64_t i = 0; i < a->n(); ++i) A2.push_back((float)(-exp((double)a->at(i)) * 1.4426950408889634));
  mb.A2 = pl.vec(std::move(A2));
  mb.D = pl.vec(ts.need(p + ".D", {I}));
  return KH_OK;
}

int load_latent(Plan& pl, Tensors& ts, const std::string& p, const JsonValue& v, int W, HyLatent& la) {
  la.H = size_of(v, "heads", ts.dim(p + ".sink", 0));
  la.R = size_of(v, "kv_rank", ts.dim(p + ".dkv.norm", 0));
  la.qr = size_of(v, "q_rank", ts.dim(p + ".dq", 0));
  if (la.H <= 0 || la.R <= 0 || la.qr <= 0) return KH_ERR_FORMAT;
  la.dn = size_of(v, "dim", ts.dim(p + ".uk", 0) / la.H);
  la.dv = size_of(v, "vdim", ts.dim(p + ".uv", 0) / la.H);
  la.dr = size_of(v, "rot_dim", ts.dim(p + ".dkv", 0) - la.R);
  if (la.dn <= 0 || la.dv <= 0 || la.dr < 0) return KH_ERR_FORMAT;
  la.scale = (float)v.number("scale", 1.0 / sqrt((double)(la.dn + la.dr)));
  if (const JsonValue* rot = v.get("rot")) {
    la.dims = rot->integer("dims", la.dr);
    la.base = rot->number("base", 10000.0);
  }
  if (la.dims < 0 || la.dims > la.dr || la.dims % 2 || !(la.base > 0)) return KH_ERR_FORMAT;
  la.dnp = padk(la.dn);
  la.drp = lat_pad_rot(la.dr);
  la.dvp = padk(la.dv);
  la.Rp = lat_pad_latent(la.R);
  la.qrp = padk(la.qr);
  if (!la.Rp || !la.drp) return KH_ERR_UNSUPPORTED;
  const int H = la.H;
  la.dqkv = pl.mat(la.qr + la.R + la.dr, W, padk(W));
  pl.put(la.dqkv, 0, ts.need(p + ".dq", {la.qr, W}), 0, la.qr);
  pl.put(la.dqkv, la.qr, ts.need(p + ".dkv", {la.R + la.dr, W}), 0, la.R + la.dr);
  la.uq = pl.mat(H * (la.dnp + la.drp), la.qr, la.qrp);
  la.ukT = pl.mat(H * la.Rp, la.dn, la.dnp);
  la.uk = pl.mat(H * la.dnp, la.R, la.Rp);
  la.uv = pl.mat(H * la.dvp, la.R, la.Rp);
  la.o = pl.mat(W, H * la.dvp, H * la.dvp);
  const Tensor *uq = ts.need(p + ".uq", {(int64_t)H * (la.dn + la.dr), la.qr}), *uk = ts.need(p + ".uk", {(int64_t)H * la.dn, la.R}),
               *uv = ts.need(p + ".uv", {(int64_t)H * la.dv, la.R}), *o = ts.need(p + ".o", {W, (int64_t)H * la.dv});
  for (int h = 0; h < H; ++h) {
    pl.put(la.uq, (int64_t)h * (la.dnp + la.drp), uq, (int64_t)h * (la.dn + la.dr), la.dn);
    pl.put(la.uq, (int64_t)h * (la.dnp + la.drp) + la.dnp, uq, (int64_t)h * (la.dn + la.dr) + la.dn, la.dr);
    pl.put(la.uk, (int64_t)h * la.dnp, uk, (int64_t)h * la.dn, la.dn);
    pl.put_t(la.ukT, (int64_t)h * la.Rp, uk, (int64_t)h * la.dn, la.dn);
    pl.put(la.uv, (int64_t)h * la.dvp, uv, (int64_t)h * la.dv, la.dv);
    pl.put(la.o, 0, o, 0, W, (int64_t)h * la.dv, la.dv, (int64_t)h * la.dvp);
  }
  la.qn = pl.vec(ts.need(p + ".dq.norm", {la.qr}));
  la.kvn = pl.vec(ts.need(p + ".dkv.norm", {la.R}));
  la.sink = pl.vec(ts.need(p + ".sink", {H}));
  return KH_OK;
}

// Entry of a distance table of `rows` entries that holds for distance n: one entry per distance below half of them, then
// entries of equal width in log distance up to `far`, the last one for everything beyond.
int distance_entry(int n, int rows, double far) {
  const int half = rows / 2;
  if (n < half || rows <= 1) return std::min(n, rows - 1);
  double x = log((double)n / half) / log(far / half) * (rows - half);
  if (!(x < rows)) return rows - 1;  // beyond `far`, or a degenerate far
  const double r = nearbyint(x);
  if (fabs(x - r) < 1e-9) x = r;  // a border up to rounding of the logarithms
  return std::max(0, std::min(rows - 1, half + (int)floor(x)));
}

enum HeadsFlags { HEADS_BIASES = 1, HEADS_REL = 2, HEADS_WINDOW = 4, HEADS_CHUNK = 8, HEADS_SINK = 16, HEADS_GATE = 32 };
// Attention over grouped heads with query / key norms; flags: projection biases, a learned distance bias, what mask.size
// means, a sink, an output gate.
int load_heads(Plan& pl, Tensors& ts, const std::string& p, const JsonValue& v, int W, int flags, HyHeads& a) {
  a.H = v.integer("heads", -1);
  a.G = v.integer("kv_heads", a.H);
  a.dk = size_of(v, "dim", ts.dim(p + ".q.norm", 0));
  if (a.H <= 0 || a.G <= 0 || a.H % a.G || a.dk <= 0) return KH_ERR_FORMAT;
  a.dv = size_of(v, "vdim", ts.dim(p + ".v", 0) / a.G);
  if (a.dv <= 0) return KH_ERR_FORMAT;
  if (a.dk > KH_HEADS_MAX_DIM || a.dv > KH_HEADS_MAX_DIM) return KH_ERR_UNSUPPORTED;
  a.scale = (float)v.number("scale", 1.0 / sqrt((double)a.dk));
  const JsonValue* mask = v.get("mask");
  const int size = mask ? mask->integer("size", 0) : 0;
  if (flags & (HEADS_WINDOW | HEADS_CHUNK)) {
    if (size <= 0) return KH_ERR_FORMAT;
    ((flags & HEADS_WINDOW) ? a.span.window : a.span.chunk) = size;
  }
  a.sink = (flags & HEADS_SINK) != 0;
  a.gate = (flags & HEADS_GATE) != 0;
  a.dkr = pad_to(a.dk, 16);
  a.dvr = pad_to(a.dv, 16);
  a.dkp = padk(a.dk);
  a.dvp = padk(a.dv);
  const int H = a.H, G = a.G, N = a.g_off() + (a.gate ? H * a.dvr : 0);
  a.qkvg = pl.mat(N, W, padk(W));
  std::vector<float> b;
  auto part = [&](const char* name, int at, int heads, int d, int dr, bool bias) {
    const Tensor* t = ts.need(p + name, {(int64_t)heads * d, W});
    for (int h = 0; h < heads; ++h) pl.put(a.qkvg, at + (int64_t)h * dr, t, (int64_t)h * d, d);
    std::vector<float> x((size_t)heads * dr, 0.f);
    if (bias) x = head_vec(ts.need(p + name + ".b", {(int64_t)heads * d}), heads, d, dr);
    b.insert(b.end(), x.begin(), x.end());
  };
  const bool biases = (flags & HEADS_BIASES) != 0;
  part(".q", 0, H, a.dk, a.dkr, biases);
  part(".k", a.k_off(), G, a.dk, a.dkr, biases);
  part(".v", a.v_off(), G, a.dv, a.dvr, biases);
  if (a.gate) part(".g", a.g_off(), H, a.dv, a.dvr, false);
  const int hv = H * a.dvr;
  a.o = pl.mat(W, hv, padk(hv));
  const Tensor* o = ts.need(p + ".o", {W, (int64_t)H * a.dv});
  for (int h = 0; h < H; ++h) pl.put(a.o, 0, o, 0, W, (int64_t)h * a.dv, a.dv, (int64_t)h * a.dvr);
  if (biases) {
    a.qkvg_b = pl.vec(std::move(b));
    a.o_b = pl.vec(ts.need(p + ".o.b", {W}));
  }
  a.qn = pl.vec(head_vec(ts.need(p + ".q.norm", {a.dk}), 1, a.dk, a.dkp));
  a.kn = pl.vec(head_vec(ts.need(p + ".k.norm", {a.dk}), 1, a.dk, a.dkp));
  if (flags & HEADS_REL) {
    const int rows = (int)ts.dim(p + ".rel", 0);
    const double far = v.number("bias_max", -1.0);
    if (rows <= 0 || !(far > 0)) return KH_ERR_FORMAT;
    const Tensor* rel = ts.need(p + ".rel", {rows, H});
    // by distance, up to the last entry's first distance or the farthest visible one
    std::vector<int> entry{distance_entry(0, rows, far)};
    const int most = a.span.window > 0 ? a.span.window : 1 << 20;
    while ((int)entry.size() < most && entry.back() < rows - 1) entry.push_back(distance_entry((int)entry.size(), rows, far));
    a.nbias = (int)entry.size();
    std::vector<float> t((size_t)H * a.nbias, 0.f);
    if (rel)
      for (int h = 0; h < H; ++h)
        for (int n = 0; n < a.nbias; ++n) t[(size_t)h * a.nbias + n] = rel->at((int64_t)entry[(size_t)n] * H + h) * 1.4426950408889634f;
    a.bias = pl.vec(std::move(t));
  }
  return KH_OK;
}

// dense feed-forward, SwiGLU: an expert every token takes
int load_dense(Plan& pl, Tensors& ts, const std::string& p, const JsonValue& v, int W, HyMoe& ff) {
  ff.on = true;
  ff.sff = size_of(v, "ff", ts.dim(p + ".gate", 0));
  if (ff.sff <= 0) return KH_ERR_FORMAT;
  ff.sffp = padk(ff.sff);
  ff.sgu = pl.mat(2 * ff.sffp, W, padk(W));
  put_gate_up(pl, ff.sgu, 0, ts.need(p + ".gate", {ff.sff, W}), ts.need(p + ".up", {ff.sff, W}), ff.sff);
  ff.sdown = pl.mat(W, ff.sff, ff.sffp);
  pl.put(ff.sdown, 0, ts.need(p + ".down", {W, ff.sff}), 0, W);
  return KH_OK;
}

// correction: the choice is by softmax over all outputs plus a correction; else weights are the softmax over the chosen
int load_moe(Plan& pl, Tensors& ts, const std::string& p, const JsonValue& v, int W, bool correction, HyMoe& ff) {
  if (v.text("kind") != "moe") return KH_ERR_UNSUPPORTED;
  const JsonValue *r = v.get("router"), *ex = v.get("expert"), *sh = v.get("shared");
  if (!r) return KH_ERR_FORMAT;
  ff.on = true;
  ff.E = r->integer("experts", -1);
  ff.ident = r->integer("identity", 0);
  ff.top = r->integer("top", -1);
  ff.ff = size_of(ex ? *ex : JsonValue(), "ff", ts.dim(p + ".e0.gate", 0));
  if (ff.E <= 0 || ff.ident < 0 || ff.top <= 0 || ff.top > ff.n_out() || ff.ff <= 0) return KH_ERR_FORMAT;
  if (ff.n_out() > KH_MOE_MAX_OUT || ff.top > KH_MOE_MAX_TOP) return KH_ERR_UNSUPPORTED;
  ff.ffp = padk(ff.ff);
  if (sh) {
    ff.sff = size_of(*sh, "ff", ts.dim(p + ".shared.gate", 0));
    if (ff.sff <= 0) return KH_ERR_FORMAT;
    ff.sffp = padk(ff.sff);
  }
  ff.zr = pl.mat(ff.n_out() + (sh ? 1 : 0), W, padk(W));
  pl.put(ff.zr, 0, ts.need(p + ".router", {ff.n_out(), W}), 0, ff.n_out());
  ff.over_chosen = !correction;
  if (correction) ff.corr = pl.vec(ts.need(p + ".correction", {ff.n_out()}));
  ff.gu = pl.mat(ff.E * 2 * ff.ffp, W, padk(W));
  ff.down = pl.mat(ff.E * W, ff.ff, ff.ffp);
  for (int e = 0; e < ff.E; ++e) {
    const std::string q = p + ".e" + std::to_string(e);
    put_gate_up(pl, ff.gu, (int64_t)e * 2 * ff.ffp, ts.need(q + ".gate", {ff.ff, W}), ts.need(q + ".up", {ff.ff, W}), ff.ff);
    pl.put(ff.down, (int64_t)e * W, ts.need(q + ".down", {W, ff.ff}), 0, W);
  }
  if (sh) {
    ff.sgate = true;
    pl.put(ff.zr, ff.n_out(), ts.need(p + ".shared.sg", {1, W}), 0, 1);
    ff.sgu = pl.mat(2 * ff.sffp, W, padk(W));
    put_gate_up(pl, ff.sgu, 0, ts.need(p + ".shared.gate", {ff.sff, W}), ts.need(p + ".shared.up", {ff.sff, W}), ff.sff);
    ff.sdown = pl.mat(W, ff.sff, ff.sffp);
    pl.put(ff.sdown, 0, ts.need(p + ".shared.down", {W, ff.sff}), 0, W);
  }
  return KH_OK;
}

// What every architecture has: sizes, norm constant, embedding, head, the looped range
int load_common(const JsonValue& cfg, Tensors& ts, Plan& pl, Hybrid& hy) {
  HyConfig& c = hy.c;
  c.width = size_of(cfg, "width", ts.dim("embed", 1));
  c.vocab = size_of(cfg, "vocab", ts.dim("embed", 0));
  const JsonValue *ls = cfg.get("layers"), *nm = cfg.get("norm"), *lp = cfg.get("loop");
  if (c.width <= 0 || c.vocab <= 0 || !ls || ls->kind != JsonValue::ARR || ls->arr.empty() || !nm) return KH_ERR_FORMAT;
  c.eps = (float)nm->number("eps", -1.0);
  if (!(c.eps > 0)) return KH_ERR_FORMAT;
  const int W = c.width;
  c.widthp = padk(W);
  hy.embed = pl.mat(c.vocab, W, c.widthp);
  pl.put(hy.embed, 0, ts.need("embed", {c.vocab, W}), 0, c.vocab);
  hy.head = pl.mat(c.vocab, W, c.widthp);
  pl.put(hy.head, 0, ts.need("head", {c.vocab, W}), 0, c.vocab);
  if (lp) {
    c.loop = true;
    c.loop_start = lp->integer("start", -1);
    c.loop_stop = lp->integer("stop", -1);
    c.loop_times = lp->integer("times", -1);
    if (c.loop_start < 0 || c.loop_stop <= c.loop_start || c.loop_stop > (int)ls->arr.size() || c.loop_times < 1) return KH_ERR_FORMAT;
  }
  return KH_OK;
}
int unknown_mixer(int layer, const std::string& type) {
  fprintf(stderr, "[kh] layer %d: unknown mixer '%s'\n", layer, type.c_str());
  return KH_ERR_UNSUPPORTED;
}

// Gufanex: parallel blocks with two layer norms, mixers mamba1 / latent_attention, mixture of experts, one looped range
// whose passes add the embedding output and a step vector
int load_gufanex(const JsonValue& cfg, Tensors& ts, Plan& pl, Hybrid& hy) {
  HyConfig& c = hy.c;
  int rc = load_common(cfg, ts, pl, hy);
  if (rc != KH_OK) return rc;
  const int W = c.width, L = (int)cfg.get("layers")->arr.size();
  c.cap = (float)cfg.number("logit_softcap", 0.0);
  hy.fnorm = pl.vec(ts.need("final.norm", {W}));
  hy.fnorm_b = pl.vec(ts.need("final.norm.b", {W}));
  if (c.loop) {
    std::vector<float> step((size_t)c.loop_times * c.widthp, 0.f);
    if (const Tensor* t = ts.need("loop.step", {c.loop_times, W}))
      for (int p = 0; p < c.loop_times; ++p)
        for (int i = 0; i < W; ++i) step[(size_t)p * c.widthp + i] = t->at((int64_t)p * W + i);
    hy.step = pl.vec(std::move(step));
  }
  for (int i = 0; i < L; ++i) {
    const JsonValue& v = cfg.get("layers")->arr[(size_t)i];
    const std::string p = "l" + std::to_string(i), type = v.text("type");
    const JsonValue *mx = v.get("mixer"), *ml = v.get("mlp");
    HyLayer ly;
    ly.n1 = pl.vec(ts.need(p + ".norm1", {W}));
    ly.n1b = pl.vec(ts.need(p + ".norm1.b", {W}));
    const JsonValue none;
    if (type == "mamba1") {
      ly.mixer = HY_MAMBA1;
      rc = load_mamba(pl, ts, p + ".mix", mx ? *mx : none, W, ly.mb);
    } else if (type == "latent_attention") {
      ly.mixer = HY_LATENT;
      rc = load_latent(pl, ts, p + ".mix", mx ? *mx : none, W, ly.la);
    } else {
      return unknown_mixer(i, type);
    }
    if (rc != KH_OK) return rc;
    if (ml) {
      ly.n2 = pl.vec(ts.need(p + ".norm2", {W}));
      ly.n2b = pl.vec(ts.need(p + ".norm2.b", {W}));
      if ((rc = load_moe(pl, ts, p + ".mlp", *ml, W, true, ly.ff)) != KH_OK) return rc;
    }
    hy.layers.push_back(ly);
  }
  return KH_OK;
}

// Gusorax: parallel blocks behind one RMS norm (weights around zero) with a residual multiplier, mixers attention
// (sliding window, distance bias) / attention_2 (chunks, sink, gate, biases), dense feed-forwards or clamped experts,
// scaled embeddings with learned positions, one looped range whose passes enter through a matrix
int load_gusorax(const JsonValue& cfg, Tensors& ts, Plan& pl, Hybrid& hy) {
  HyConfig& c = hy.c;
  int rc = load_common(cfg, ts, pl, hy);
  if (rc != KH_OK) return rc;
  const int W = c.width, L = (int)cfg.get("layers")->arr.size();
  c.rms = true;
  c.mult = (float)cfg.number("residual_mult", 1.0);
  if (const JsonValue* e = cfg.get("embedding")) c.emb_scale = (float)e->number("scale", 1.0);
  c.max_pos = size_of(cfg, "max_positions", ts.dim("pos", 0));
  if (c.max_pos <= 0) return KH_ERR_FORMAT;
  hy.pos_emb = pl.mat(c.max_pos, W, c.widthp);
  pl.put(hy.pos_emb, 0, ts.need("pos", {c.max_pos, W}), 0, c.max_pos);
  auto norm = [&](const std::string& name) {
    std::vector<float> v = head_vec(ts.need(name, {W}), 1, W, W);
    for (float& x : v) x += 1.f;
    return pl.vec(std::move(v));
  };
  hy.fnorm = norm("final.norm");
  if (c.loop) {
    const Tensor* t = ts.need("loop.in", {W, 2 * W});
    hy.enter = pl.mat(W, 2 * c.widthp, 2 * c.widthp);
    pl.put(hy.enter, 0, t, 0, W, 0, W, 0);
    pl.put(hy.enter, 0, t, 0, W, W, W, c.widthp);
  }
  for (int i = 0; i < L; ++i) {
    const JsonValue& v = cfg.get("layers")->arr[(size_t)i];
    const std::string p = "l" + std::to_string(i), type = v.text("type");
    const JsonValue *mx = v.get("mixer"), *ml = v.get("mlp");
    HyLayer ly;
    ly.n1 = norm(p + ".norm1");
    int flags;
    if (type == "attention") flags = HEADS_REL | HEADS_WINDOW;
    else if (type == "attention_2") flags = HEADS_BIASES | HEADS_CHUNK | HEADS_SINK | HEADS_GATE;
    else return unknown_mixer(i, type);
    if (!mx) return KH_ERR_FORMAT;
    ly.mixer = HY_HEADS;
    if ((rc = load_heads(pl, ts, p + ".mix", *mx, W, flags, ly.ha)) != KH_OK) return rc;
    if (ml && ml->text("kind") == "dense") {
      if ((rc = load_dense(pl, ts, p + ".mlp", *ml, W, ly.ff)) != KH_OK) return rc;
    } else if (ml) {
      if ((rc = load_moe(pl, ts, p + ".mlp", *ml, W, false, ly.ff)) != KH_OK) return rc;
      const JsonValue* ex = ml->get("expert");
      ly.ff.act = GateAct{(float)(ex ? ex->number("limit", INFINITY) : INFINITY), 1.702f, 1.f};
    }
    hy.layers.push_back(ly);
  }
  return KH_OK;
}

struct Arch {
  const char* name;
  int (*load)(const JsonValue&, Tensors&, Plan&, Hybrid&);
};
const Arch kArchs[] = {{"Gufanex", load_gufanex}, {"Gusorax", load_gusorax}};

// runs in execution order, and where each finds its part of a slot's state
void build_runs(Hybrid& hy) {
  const HyConfig& c = hy.c;
  const int L = (int)hy.layers.size();
  auto add = [&](int l, int pass) {
    HyRun r;
    r.layer = l;
    r.pass = pass;
    hy.runs.push_back(r);
  };
  const int s = c.loop ? c.loop_start : L, e = c.loop ? c.loop_stop : L;
  for (int l = 0; l < s; ++l) add(l, -1);
  if (c.loop)
    for (int t = 0; t < c.loop_times; ++t)
      for (int l = s; l < e; ++l) add(l, l == s ? t : -1);
  for (int l = e; l < L; ++l) add(l, -1);
}

template <class F>
void each_mat(Hybrid& hy, F&& f) {
  for (HyMat* m : {&hy.embed, &hy.head, &hy.pos_emb, &hy.enter})
    if (m->N) f(*m);
  for (auto& l : hy.layers) {
    for (HyMat* m : {&l.mb.in, &l.mb.x, &l.mb.dt, &l.mb.o, &l.la.dqkv, &l.la.uq, &l.la.ukT, &l.la.uk, &l.la.uv, &l.la.o, &l.ha.qkvg,
                     &l.ha.o, &l.ff.zr, &l.ff.gu, &l.ff.down, &l.ff.sgu, &l.ff.sdown})
      if (m->N) f(*m);
  }
}
template <class F>
void each_vec(Hybrid& hy, F&& f) {
  for (HyVec* v : {&hy.fnorm, &hy.fnorm_b, &hy.step})
    if (v->on) f(*v);
  for (auto& l : hy.layers)
    for (HyVec* v : {&l.n1, &l.n1b, &l.n2, &l.n2b, &l.mb.conv, &l.mb.conv_b, &l.mb.dt_b, &l.mb.A2, &l.mb.D, &l.la.qn,
                     &l.la.kvn, &l.la.sink, &l.ha.qkvg_b, &l.ha.o_b, &l.ha.qn, &l.ha.kn, &l.ha.bias, &l.ff.corr})
      if (v->on) f(*v);
}

// cache rows a run of the layer keeps per sequence
int cache_rows(const HyLayer& l, int cache_len) { return l.mixer == HY_HEADS ? l.ha.ring : cache_len; }

int alloc_workspace(kh_model* m) {
  Hybrid& hy = *m->hy;
  const size_t T = (size_t)hy.tmax, Wp = (size_t)hy.c.widthp, es = hy.elem();
  size_t f32a = 1, a0 = 1, a1 = 1, a2 = 1, dt = 1, bc = 1, z = 1, ends = 1, dtsum = 1, h = 1, hs = 1, y = 1, top = 1, tiles = 1;
  auto up = [](size_t& v, size_t n) { v = v > n ? v : n; };
  const size_t multi = T / KH_SCAN_CH * 2 + 2;  // chunks of segments that have more than one
  if (hy.enter.N) up(a2, T * 2 * Wp);
  for (auto& l : hy.layers) {
    if (l.mixer == HY_MAMBA1) {
      const size_t I = (size_t)l.mb.inner, Ip = (size_t)l.mb.innerp;
      up(a0, T * 2 * I);
      up(a1, T * Ip);
      up(a2, T * Ip);
      up(a2, T * (size_t)l.mb.rankp);
      up(dt, T * I);
      up(bc, T * 2 * (size_t)l.mb.state);
      up(ends, multi * I * (size_t)l.mb.state);
      up(dtsum, multi * I);
    } else if (l.mixer == HY_HEADS) {
      up(a1, T * (size_t)l.ha.qkvg.N);
      up(a0, T * (size_t)l.ha.o.ld);
    } else {
      const HyLatent& a = l.la;
      up(f32a, T * (size_t)(a.qr + a.R + a.dr));
      up(a0, T * (size_t)(a.qrp));
      up(a0, T * (size_t)(a.H * a.Rp));
      up(a0, T * (size_t)(a.H * a.dvp));
      hy.any_latent = true;
      up(a1, T * (size_t)(a.H * (a.dnp + a.drp)));
      up(a1, T * (size_t)(a.H * a.dvp));
      up(a2, T * (size_t)(a.H * a.row()));
    }
    if (l.ff.on) {
      const HyMoe& f = l.ff;
      up(z, T * (size_t)f.zr.N);
      up(h, T * (size_t)f.top * (size_t)f.ffp);
      up(y, T * (size_t)f.top * Wp);
      up(top, (size_t)f.top);
      up(hs, T * (size_t)f.sffp);
      up(tiles, T * (size_t)f.top / 32 + (size_t)f.E + 1);
    }
  }
  int rc;
  auto zf = [&](float** p, size_t n) -> int {
    if ((rc = dalloc(p, n)) != KH_OK) return rc;
    return (int)hipMemsetAsync(*p, 0, n * 4, m->stream);
  };
  auto zt = [&](void** p, size_t n) -> int {  // operand buffers: every element must be finite, also the pads
    if ((rc = dalloc((char**)p, n * es)) != KH_OK) return rc;
    return (int)hipMemsetAsync(*p, 0, n * es, m->stream);
  };
  auto zi = [&](int32_t** p, size_t n) -> int {
    if ((rc = dalloc(p, n)) != KH_OK) return rc;
    return (int)hipMemsetAsync(*p, 0, n * 4, m->stream);
  };
#define TRY(e) \
  if ((rc = (e)) != KH_OK) return rc
  TRY(zf(&hy.x, T * Wp));
  TRY(zf(&hy.x0, T * Wp));
  TRY(zf(&hy.mix, T * Wp));
  TRY(zt((void**)&hy.sh, T * Wp));
  TRY(zf(&hy.f32a, f32a));
  TRY(zf(&hy.dt, dt));
  TRY(zf(&hy.bc, bc));
  TRY(zf(&hy.z, z));
  TRY(zf(&hy.ends, ends));
  TRY(zf(&hy.dtsum, dtsum));
  TRY(zt((void**)&hy.y, y));
  TRY(zf(&hy.moe_w, T * top));
  TRY(zf(&hy.id_w, T));
  TRY(zf(&hy.sh_g, T));
  TRY(zt(&hy.xn1, T * Wp));
  TRY(zt(&hy.xn2, T * Wp));
  TRY(zt(&hy.a0, a0));
  TRY(zt(&hy.a1, a1));
  TRY(zt(&hy.a2, a2));
  TRY(zt(&hy.h, h));
  TRY(zt(&hy.hs, hs));
  TRY(zi(&hy.moe_id, T * top));
  TRY(zi(&hy.moe_rows, T * top));
  TRY(zi(&hy.moe_slot, T * top));
  TRY(zi(&hy.n_tiles, 1));
  TRY(zi((int32_t**)&hy.tiles, tiles * 4));
  hy.max_tiles = (int)tiles;
  hy.wl_rows = 64;
  TRY(zt(&hy.xw, (size_t)hy.wl_rows * Wp));
  TRY(zf(&hy.wlogits, (size_t)hy.wl_rows * hy.c.vocab));
#undef TRY
  return KH_OK;
}

int finish(kh_model* m, Plan& pl) {
  Hybrid& hy = *m->hy;
  int rc;
  const size_t bytes = pl.elems * hy.elem();
  {
    std::vector<char> img(bytes, 0);
    pl.run(hy.f32, img.data());
    KH_CHECK_HIP(hipMalloc((void**)&m->arena, bytes));
    m->owns_arena = true;
    m->arena_bytes = bytes;
    m->cfg.weight_bytes = (int64_t)bytes;
    KH_CHECK_HIP(upload_chunked(m->arena, img.data(), bytes, m->stream, &m->load_ms));
  }
  {
    std::vector<float> f((pl.floats + 127) / 64 * 64, 0.f);  // vectors are read in whole padded rows
    for (auto& v : pl.vecs) memcpy(f.data() + v.first, v.second.data(), v.second.size() * 4);
    KH_CHECK_HIP(hipMalloc((void**)&hy.farena, f.size() * 4));
    KH_CHECK_HIP(hipMemcpy(hy.farena, f.data(), f.size() * 4, hipMemcpyHostToDevice));
  }
  each_mat(hy, [&](HyMat& x) { x.w = m->arena + x.off * hy.elem(); });
  each_vec(hy, [&](HyVec& x) { x.p = (const float*)hy.farena + x.off; });
  // rotation tables, one per (base, dims)
  const int CL = m->cfg.cache_len;
  std::map<std::pair<double, int>, float2*> tabs;
  for (auto& l : hy.layers) {
    if (l.mixer != HY_LATENT || l.la.dims == 0) continue;
    float2*& d = tabs[{l.la.base, l.la.dims}];
    if (!d) {
      const int half = l.la.dims / 2;
      std::vector<float2> t((size_t)CL * half);
      for (int i = 0; i < half; ++i) {
        const double f = pow(l.la.base, -2.0 * i / l.la.dims);
        for (int p = 0; p < CL; ++p) t[(size_t)p * half + i] = float2{(float)cos(p * f), (float)sin(p * f)};
      }
      KH_CHECK_HIP(hipMalloc((void**)&d, t.size() * sizeof(float2)));
      hy.rope_tabs.push_back(d);
      KH_CHECK_HIP(hipMemcpy(d, t.data(), t.size() * sizeof(float2), hipMemcpyHostToDevice));
    }
    l.la.rope = d;
  }
  // ---- state manager
  const char* tm = dbg("KH_HY_TMAX");
  hy.tmax = tm ? std::max(32, std::min(atoi(tm), KH_HY_TMAX)) : KH_HY_TMAX;
  for (auto& l : hy.layers) {
    if (l.mixer != HY_HEADS) continue;
    HyHeads& a = l.ha;
    // a query's span and the tokens of one pass, which are all written before the first of them attends
    const int span = a.span.window > 0 ? a.span.window : a.span.chunk;
    a.ring = span > 0 && span < CL - hy.tmax ? std::min(CL, pad_to(span + hy.tmax, 64)) : CL;
    // time splits of a decoded token: tiles of the visible keys over about two workgroups per CU
    const int keys = span > 0 ? std::min(span, CL) : CL;
    a.nsplit = 2;
    while (a.nsplit < 128 && a.nsplit * KH_LAT_SPLIT_MIN < keys && a.nsplit * a.G < 512) a.nsplit *= 2;
    if ((double)a.ring * a.row() * hy.elem() >= 4294967296.0) return KH_ERR_UNSUPPORTED;  // 32-bit offsets within a run
  }
  build_runs(hy);
  for (auto& r : hy.runs) {
    const HyLayer& l = hy.layers[(size_t)r.layer];
    if (l.mixer == HY_MAMBA1) {
      r.st_off = hy.st_slot;
      hy.st_slot += ((size_t)l.mb.inner * l.mb.state + 63) / 64 * 64;
      r.conv_off = hy.st_slot;
      hy.st_slot += ((size_t)l.mb.inner * (l.mb.taps - 1) + 63) / 64 * 64;
    } else {
      r.kv_off = hy.kv_slot;
      hy.kv_slot += (size_t)cache_rows(l, CL) * l.cache_row();
    }
  }
  hy.len.assign((size_t)hy.slots, -1);
  hy.rows_ok.assign((size_t)hy.slots, 0);
  if ((rc = dalloc(&hy.state, hy.st_slot * hy.slots + 64)) != KH_OK) return rc;
  KH_CHECK_HIP(hipMemsetAsync(hy.state, 0, (hy.st_slot * hy.slots + 64) * 4, m->stream));
  if (hy.kv_slot)
    if ((rc = kv_allocate_bytes(m, hy.kv_slot * hy.slots * hy.elem(), 1)) != KH_OK) return rc;
  if ((rc = alloc_workspace(m)) != KH_OK) return rc;
  // common buffers of the model level
  if ((rc = dalloc(&m->logits, (size_t)hy.c.vocab)) != KH_OK) return rc;
  for (int32_t** p : {&m->d_pos, &m->d_token, &m->d_next})
    if ((rc = dalloc(p, 1)) != KH_OK) return rc;
  KH_CHECK_HIP(hipMemsetAsync(m->d_pos, 0, 4, m->stream));
  KH_CHECK_HIP(hipMemsetAsync(m->d_token, 0, 4, m->stream));
  KH_CHECK_HIP(hipEventCreate(&m->ev0));
  KH_CHECK_HIP(hipEventCreate(&m->ev1));
  if ((rc = ensure_seq_cap(m, 256)) != KH_OK) return rc;
  if ((rc = hy_step_init(m)) != KH_OK) return rc;
  // one eager step (token 0 at position 0 of slot 0, which every sequence starts by overwriting): kernel attributes and
  // the one-token tables exist before a step is ever captured
  if ((rc = hy_kv_ensure(m, 0, 1)) != KH_OK) return rc;
  hy_launch_step(m, 0, 0);
  if ((rc = kh_launch_status()) != KH_OK) return rc;
  KH_CHECK_HIP(hipStreamSynchronize(m->stream));
  return KH_OK;
}

int create_impl(const char* config, size_t config_len, const void* tensors, size_t nbytes, const kh_model_opts* o,
                kh_model** out) {
  int ndev = 0;
  if (hipGetDeviceCount(&ndev) != hipSuccess || ndev <= 0) {
    (void)hipGetLastError();
    return KH_ERR_NO_DEVICE;
  }
  if (o->device < 0 || o->device >= ndev || o->max_seqs < 0 || o->max_seq_len < 0) return KH_ERR_INVALID_ARG;
  if (o->dtype != KH_DTYPE_DEFAULT && o->dtype != KH_DTYPE_BF16 && o->dtype != KH_DTYPE_F32) return KH_ERR_INVALID_ARG;
  if (o->is_quant) return KH_ERR_UNSUPPORTED;
  Json j{config, config + config_len};
  JsonValue cfg;
  if (!json_parse(j, &cfg) || cfg.kind != JsonValue::OBJ) return KH_ERR_FORMAT;
  const std::string arch = cfg.text("architecture");
  const Arch* ar = nullptr;
  for (const Arch& a : kArchs)
    if (arch == a.name) ar = &a;
  if (!ar) {
    fprintf(stderr, "[kh] config.json: unknown architecture '%s'\n", arch.c_str());
    return KH_ERR_UNSUPPORTED;
  }
  Tensors ts;
  int rc = ts.parse((const char*)tensors, nbytes);
  if (rc != KH_OK) return rc;
  std::unique_ptr<Hybrid> hy(new Hybrid());
  Plan pl;
  hy->c.arch = arch;
  hy->f32 = o->dtype == KH_DTYPE_F32;
  hy->slots = o->max_seqs > 0 ? o->max_seqs : 1;
  if ((rc = ar->load(cfg, ts, pl, *hy)) != KH_OK) return rc;
  if (!ts.missing.empty()) {
    fprintf(stderr, "[kh] model.safetensors: '%s' is missing or has an unexpected shape\n", ts.missing.c_str());
    return KH_ERR_FORMAT;
  }
  KH_CHECK_HIP(hipSetDevice(o->device));
  kh_model* m = new kh_model();
  m->opts = *o;
  m->opts.family = KH_FAMILY_LAYERS;
  m->hy = hy.release();
  *out = m;
  KH_CHECK_HIP(hipStreamCreateWithFlags(&m->stream, hipStreamNonBlocking));
  kh_config& c = m->cfg;
  const Hybrid& h = *m->hy;
  c.dim = h.c.width;
  c.vocab_size = h.c.vocab;
  c.layer_num = (int)h.layers.size();
  c.family = KH_FAMILY_LAYERS;
  c.rms_eps = h.c.eps;
  c.cache_len = c.seq_len = o->max_seq_len > 0 ? o->max_seq_len : 8192;
  if (h.c.max_pos > 0 && c.cache_len > h.c.max_pos) c.cache_len = c.seq_len = h.c.max_pos;
  c.kv_mul = 1;
  for (auto& l : h.layers) {
    if (l.mixer == HY_LATENT) {
      c.head_num = c.kv_head_num = l.la.H;
      c.kv_dim = l.la.R + l.la.dr;
      c.head_size = l.la.dn + l.la.dr;
      c.rope_theta = (float)l.la.base;
    } else if (l.mixer == HY_HEADS) {
      c.head_num = l.ha.H;
      c.kv_head_num = l.ha.G;
      c.kv_dim = l.ha.G * l.ha.dk;
      c.kv_mul = l.ha.H / l.ha.G;
      c.head_size = l.ha.dk;
    }
    if (l.ff.on) c.hidden_dim = l.ff.top ? l.ff.ff : l.ff.sff;
  }
  return finish(m, pl);
}

}  // namespace

namespace khm {
int hy_create(const char* config, size_t config_len, const void* tensors, size_t nbytes, const kh_model_opts* o,
              kh_model** out) {
  *out = nullptr;
  const int rc = kh_api_guard([&] { return create_impl(config, config_len, tensors, nbytes, o, out); });
  if (rc != KH_OK && *out) {
    kh_model_destroy(*out);
    *out = nullptr;
  }
  return rc;
}

void hy_destroy(kh_model* m) {
  Hybrid* h = m->hy;
  if (!h) return;
  void* dev[] = {h->farena, h->state, h->x, h->x0, h->mix, h->f32a, h->y, h->sh, h->dt, h->bc, h->z, h->ends, h->dtsum,
                 h->moe_w, h->id_w, h->sh_g, h->wlogits, h->xn1, h->xn2, h->a0, h->a1, h->a2, h->h, h->hs, h->xw,
                 h->moe_id, h->moe_rows, h->moe_slot, h->n_tiles, h->tiles, h->kx, h->vx, h->d_tab, h->d_one};
  for (void* p : dev)
    if (p) (void)hipFree(p);
  for (float2* t : h->rope_tabs) (void)hipFree(t);
  if (h->h_tab) (void)hipHostFree(h->h_tab);
  delete h;
  m->hy = nullptr;
}

int hy_kv_ensure(kh_model* m, int slot, int rows) {
  Hybrid& hy = *m->hy;
  if (rows <= hy.rows_ok[(size_t)slot] || !hy.kv_slot) return KH_OK;
  for (const HyRun& r : hy.runs) {
    const HyLayer& l = hy.layers[(size_t)r.layer];
    if (!l.cache_row()) continue;
    const size_t row_b = (size_t)l.cache_row() * hy.elem();
    const size_t b0 = ((size_t)slot * hy.kv_slot + r.kv_off) * hy.elem();
    const int rc = kv_map_range(m, 0, b0, b0 + (size_t)std::min(rows, cache_rows(l, m->cfg.cache_len)) * row_b, r.layer);
    if (rc != KH_OK) return rc;
  }
  hy.rows_ok[(size_t)slot] = rows;
  return KH_OK;
}

int hy_expand_buffers(kh_model* m, int keys) {
  Hybrid& hy = *m->hy;
  size_t k = 0, v = 0;
  const size_t n = (size_t)pad_to(keys, 512);
  for (auto& l : hy.layers)
    if (l.mixer == HY_LATENT) {
      k = std::max(k, n * l.la.H * l.la.dnp);
      v = std::max(v, n * l.la.H * l.la.dvp);
    }
  for (void** p : {&hy.kx, &hy.vx}) {
    if (*p) (void)hipFree(*p);
    *p = nullptr;
  }
  hy.exp_keys = 0;
  int rc;
  if ((rc = dalloc((char**)&hy.kx, k * hy.elem())) != KH_OK) return rc;
  if ((rc = dalloc((char**)&hy.vx, v * hy.elem())) != KH_OK) return rc;
  // columns behind a sequence's last key are read as operands under zero weights: they must be finite
  KH_CHECK_HIP(hipMemsetAsync(hy.kx, 0, k * hy.elem(), m->stream));
  KH_CHECK_HIP(hipMemsetAsync(hy.vx, 0, v * hy.elem(), m->stream));
  hy.exp_keys = (int)n;
  return KH_OK;
}

bool hy_is_folder(const char* path) {
  struct stat st;
  return stat(path, &st) == 0 && S_ISDIR(st.st_mode);
}
int hy_create_from_folder(const char* path, const kh_model_opts* o, kh_model** out) {
  struct Map {
    void* p = nullptr;
    size_t n = 0;
    int open_file(const std::string& f) {
      const int fd = open(f.c_str(), O_RDONLY);
      if (fd < 0) return KH_ERR_IO;
      struct stat st;
      if (fstat(fd, &st) != 0 || st.st_size <= 0) {
        close(fd);
        return KH_ERR_IO;
      }
      n = (size_t)st.st_size;
      p = mmap(nullptr, n, PROT_READ, MAP_PRIVATE, fd, 0);
      close(fd);
      if (p == MAP_FAILED) {
        p = nullptr;
        return KH_ERR_IO;
      }
      return KH_OK;
    }
    ~Map() {
      if (p) munmap(p, n);
    }
  } cfg, st;
  int rc;
  if ((rc = cfg.open_file(std::string(path) + "/config.json")) != KH_OK) return rc;
  if ((rc = st.open_file(std::string(path) + "/model.safetensors")) != KH_OK) return rc;
  return hy_create((const char*)cfg.p, cfg.n, st.p, st.n, o, out);
}
}  // namespace khm

extern "C" int kh_model_create_from_checkpoint(const char* h_config_json, size_t config_len, const void* h_safetensors,
                                               size_t nbytes, const kh_model_opts* opts, kh_model** out) {
  if (!h_config_json || !h_safetensors || !opts || !out) return KH_ERR_INVALID_ARG;
  return hy_create(h_config_json, config_len, h_safetensors, nbytes, opts, out);
}
