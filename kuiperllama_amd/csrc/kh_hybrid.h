// kh_hybrid.h — host-side description of a layer-list model (a checkpoint folder: config.json + model.safetensors):
// a list of layers, each with one of several mixers and one of several feed-forwards of its own sizes, a block of
// layers that may run several times, and the state its sequences carry.  Attached to kh_model::hy; the C-ABI entry
// points of the model level dispatch on it.
//   kh_hybrid_load.hip   config + weights -> HBM arena, state manager
//   kh_hybrid_pass.hip   a pass of T tokens of several sequences on the matrix cores (prompts, mixed lengths)
//   kh_hybrid_step.hip   the fused decode step, batches, C-ABI
#pragma once
#include <memory>
#include <string>
#include <vector>

#include "kh_heads.h"
#include "kh_json.h"
#include "kh_latent.h"
#include "kh_lgemm.h"
#include "kh_model_internal.h"
#include "kh_moe.h"
#include "kh_scan.h"

#define KH_HY_TMAX 2048       // tokens of one pass
#define KH_HY_DECODE_B 4      // sequences of one fused decode step, at most

namespace khm {

// rows [N][ld] of storage type T in the arena
struct HyMat {
  size_t off = 0;  // element offset in the arena (load time)
  const void* w = nullptr;
  int N = 0, K = 0, ld = 0;
};
struct HyVec {  // fp32 parameters
  size_t off = 0;
  const float* p = nullptr;  // nullptr: the model has none
  bool on = false;
};

enum HyMixer { HY_MAMBA1 = 0, HY_LATENT = 1, HY_HEADS = 2 };

struct HyMamba {
  int inner = 0, state = 0, rank = 0, taps = 0;
  int innerp = 0, rankp = 0;
  HyMat in, x, dt, o;  // x: rows [dt rank (padded to rankp) | B | C]
  HyVec conv, conv_b, dt_b, A2, D;
};
struct HyLatent {
  int H = 0, dn = 0, dr = 0, dv = 0, R = 0, qr = 0, dims = 0;
  int dnp = 0, drp = 0, dvp = 0, Rp = 0, qrp = 0;
  float scale = 1.f;
  double base = 10000.0;
  HyMat dqkv;  // [q latent | kv latent | rotated key part]
  HyMat uq;    // head by head [dnp | drp]
  HyMat ukT;   // head by head [Rp][dnp]: W_uk transposed
  HyMat uk;    // head by head [dnp][Rp]
  HyMat uv;    // head by head [dvp][Rp]
  HyMat o;     // columns head by head, dvp each
  HyVec qn, kvn, sink;
  const float2* rope = nullptr;
  int row() const { return Rp + drp; }
};
struct HyHeads {  // attention over cached keys and values, grouped heads
  int H = 0, G = 0, dk = 0, dv = 0;
  int dkr = 0, dvr = 0;  // rows of a projected head (multiples of 16)
  int dkp = 0, dvp = 0;  // elements of a cached head (multiples of 64)
  float scale = 1.f;
  KeySpan span{0, 0};
  int nbias = 0, ring = 0, nsplit = 1;
  bool gate = false, sink = false;
  HyMat qkvg;  // query heads, key heads, value heads, gate rows
  HyMat o;     // columns head by head, dvr each
  HyVec qkvg_b, o_b, qn, kn, bias;
  int row() const { return G * (dkp + dvp); }
  int k_off() const { return H * dkr; }
  int v_off() const { return k_off() + G * dkr; }
  int g_off() const { return v_off() + G * dvr; }
  HeadRow head_row(float eps) const { return {kn.p, G, dk, dv, dkr, dvr, dkp, dvp, k_off(), v_off(), ring, eps}; }
};
// Feed-forward: routed experts and / or one every token takes (a dense feed-forward is the latter alone)
struct HyMoe {
  bool on = false, over_chosen = false;
  int E = 0, ident = 0, top = 0, ff = 0, ffp = 0, sff = 0, sffp = 0;  // top 0: no router; sff 0: no shared expert
  bool sgate = false;  // the shared expert has a gate row
  GateAct act{INFINITY, 1.f, 0.f}, sact{INFINITY, 1.f, 0.f};
  HyMat zr;    // router rows, then the shared expert's gate row
  HyMat gu;    // experts, each [2 ffp]: 16 gate rows, 16 up rows, ...
  HyMat down;  // experts, each [W][ffp]
  HyMat sgu, sdown;
  HyVec corr;
  int n_out() const { return E + ident; }
};
struct HyLayer {
  int mixer = HY_MAMBA1;
  HyMamba mb;
  HyLatent la;
  HyHeads ha;
  HyMoe ff;
  HyVec n1, n1b, n2, n2b;  // n2 off: the feed-forward reads the first norm
  const HyMat& out_mat() const { return mixer == HY_MAMBA1 ? mb.o : (mixer == HY_LATENT ? la.o : ha.o); }
  const HyVec& norm2() const { return n2.on ? n2 : n1; }
  const HyVec& norm2_b() const { return n2.on ? n2b : n1b; }
  int cache_row() const { return mixer == HY_LATENT ? la.row() : (mixer == HY_HEADS ? ha.row() : 0); }  // elements
};
// one run of a layer: a looped layer has one per pass, each with its own cache or state
struct HyRun {
  int layer = 0;
  int pass = -1;   // >= 0: first layer of pass `pass` of the loop
  size_t st_off = 0, conv_off = 0;  // mamba: floats within a slot's state
  size_t kv_off = 0;                // attention: elements within a slot's cache range
};
struct HyConfig {
  std::string arch;
  int width = 0, vocab = 0, widthp = 0;
  float eps = 1e-5f, cap = 0.f, mult = 1.f, emb_scale = 1.f;
  bool rms = false;    // RMS norms without biases (else layer norms)
  int max_pos = 0;     // positions the model has (0: any)
  int loop_start = 0, loop_stop = 0, loop_times = 1;
  bool loop = false;
};

struct Hybrid {
  HyConfig c;
  bool f32 = false;  // storage type: fp32 instead of bf16
  std::vector<HyLayer> layers;
  std::vector<HyRun> runs;
  HyMat embed, head, pos_emb;
  HyMat enter;  // a pass of the loop starts with x <- enter [x ; embedding output]
  HyVec fnorm, fnorm_b, step;
  char* farena = nullptr;  // fp32 parameters
  std::vector<float2*> rope_tabs;
  size_t elem() const { return f32 ? 4 : 2; }

  // ---- sequences: slot s owns state floats [s * st_slot, ...) and cache elements [s * kv_slot, ...)
  int slots = 1;
  std::vector<int> len;        // tokens a slot holds; -1: free
  std::vector<int> rows_ok;    // cache rows of a slot that are backed by memory
  size_t st_slot = 0, kv_slot = 0;
  float* state = nullptr;
  // ---- pass workspace (allocated at creation for KH_HY_TMAX tokens)
  int tmax = 0;
  float *x = nullptr, *x0 = nullptr, *mix = nullptr, *f32a = nullptr, *y = nullptr, *sh = nullptr, *dt = nullptr,
        *bc = nullptr, *z = nullptr, *ends = nullptr, *dtsum = nullptr, *moe_w = nullptr, *id_w = nullptr,
        *sh_g = nullptr, *wlogits = nullptr;
  void *xn1 = nullptr, *xn2 = nullptr, *a0 = nullptr, *a1 = nullptr, *a2 = nullptr, *h = nullptr, *hs = nullptr,
       *xw = nullptr;
  // expanded latent attention: keys [exp_keys][H dnp] and transposed values [H dvp][exp_keys] of one segment
  void *kx = nullptr, *vx = nullptr;
  int exp_keys = 0;
  bool any_latent = false;
  int32_t *moe_id = nullptr, *moe_rows = nullptr, *moe_slot = nullptr, *n_tiles = nullptr;
  LgTile* tiles = nullptr;
  int max_tiles = 0;
  int wl_rows = 0;        // rows wlogits / xw hold
  // pass tables: pinned staging and device copy
  int32_t *h_tab = nullptr, *d_tab = nullptr;
  size_t tab_cap = 0;
  // one-token tables of the decode step (device-resident, written by k_one_tabs)
  int32_t* d_one = nullptr;
  // ---- decode step
  struct Step;
  std::unique_ptr<Step> step_st;
  // residual probe: after every layer run the pass appends x [T][W] here
  float* probe = nullptr;
  int64_t probe_cap = 0, probe_n = 0;
  Hybrid();
  ~Hybrid();
};

struct HyEntry {  // tokens of one sequence in a pass
  int slot, n, pos0;
  const int32_t* tok;
};

// the attention arguments that follow from the model; the caller adds rows, output and splits
inline HeadsArgs heads_args(const Hybrid& hy, const HyHeads& a, const void* cache) {
  HeadsArgs h{};
  h.g_off = a.gate ? a.g_off() : -1;
  h.qn = a.qn.p;
  h.cache = cache;
  h.slot_elems = hy.kv_slot;
  h.bias = a.bias.p;
  h.H = a.H;
  h.G = a.G;
  h.dk = a.dk;
  h.dkr = a.dkr;
  h.dkp = a.dkp;
  h.dvr = a.dvr;
  h.dvp = a.dvp;
  h.ring = a.ring;
  h.nsplit = 1;
  h.nbias = a.nbias;
  h.sink = a.sink;
  h.span = a.span;
  h.eps = hy.c.eps;
  h.scale2 = a.scale * 1.44269504088896f;
  return h;
}

// ---- kh_hybrid_load.hip
int hy_create(const char* config, size_t config_len, const void* tensors, size_t nbytes, const kh_model_opts* o, kh_model** out);
void hy_destroy(kh_model* m);
int hy_expand_buffers(kh_model* m, int keys);       // room for the expanded keys / values of that many tokens
int hy_kv_ensure(kh_model* m, int slot, int rows);  // cache rows [0, rows) of a slot backed by memory
bool hy_is_folder(const char* path);
int hy_create_from_folder(const char* path, const kh_model_opts* o, kh_model** out);
// ---- kh_hybrid_pass.hip
// Runs the entries' tokens (any mixture of lengths, cut into passes as needed).  want: rows of the concatenated tokens
// whose logits are wanted (ascending); they arrive in h_logits.  Returns after the stream has drained when h_logits.
int hy_forward(kh_model* m, const HyEntry* e, int n, const int32_t* want, int n_want, float* h_logits);
// one token at (d_token, d_pos) of slot 0 on the pass kernels, logits to m->logits (the unfused step)
int hy_unfused_step(kh_model* m);
// argmax of m->logits as one sampler partial
int hy_argmax_partial(kh_model* m);
// ---- kh_hybrid_step.hip
int hy_step_init(kh_model* m);
void hy_launch_step(kh_model* m, int advance, int n_forced);
int hy_decode_max(const kh_model* m);  // sequences the fused step can take at once
int hy_decode(kh_model* m, const HyEntry* e, int n, float* h_logits);
int hy_launches(const kh_model* m);  // kernel launches of one decode step
}  // namespace khm
