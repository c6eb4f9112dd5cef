// kh_hybrid_step.hip — layer-list models: the decode step of the generate loop, sequence slots, batches.
#include <string.h>

#include <algorithm>

#include "kh_fused.h"
#include "kh_hybrid.h"

using namespace khm;

namespace khm {
struct Hybrid::Step {
  int dummy = 0;
};
Hybrid::Hybrid() {}
Hybrid::~Hybrid() {}

int hy_step_init(kh_model* m) {
  (void)m;
  return KH_OK;
}
void hy_launch_step(kh_model* m, int advance, int n_forced) {
  (void)hy_unfused_step(m);
  (void)kh_argmax_f32(m->logits, m->cfg.vocab_size, m->d_next, (void*)m->stream);
  (void)advance; (void)n_forced;
}
int hy_launches(const kh_model* m) { return (int)m->hy->runs.size() * 15; }
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
  if ((rc = hy_forward(m, es.data(), n, want.data(), (int)want.size(), want.empty() ? nullptr : h_logits)) != KH_OK) return rc;
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
