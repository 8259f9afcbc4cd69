// Continuous batching over a decoder's sequences: requests wait, are admitted when a sequence and enough cache are free, bring
// their prompt in portions beside the single tokens of the requests that already decode, and give everything back when they are
// finished.  One scheduler step is one cai_decoder_step_batch.  Host code only.
#include "cai_layered.hpp"

#include <algorithm>
#include <deque>
#include <map>
#include <memory>

using namespace cai;

namespace {

struct Request {
  int64_t id = 0;
  std::vector<int32_t> prompt, out;
  size_t fed = 0;                          // prompt tokens already in the cache
  int max_new = 0, eos = -1, top_k = 0; float temperature = 0.0f; uint64_t rng = 0;
  int seq = -1, pages = 0; bool done = false;

  double draw()                            // uniform in [0, 1): splitmix64
  {
    uint64_t z = (rng += 0x9e3779b97f4a7c15ull);
    z = (z ^ (z >> 30)) * 0xbf58476d1ce4e5b9ull; z = (z ^ (z >> 27)) * 0x94d049bb133111ebull; z ^= z >> 31;
    return (double)(z >> 11) * (1.0 / 9007199254740992.0);
  }
};

}  // namespace

struct cai_sched_s {
  cai_decoder_s* d = nullptr;
  cai_decoder_config cfg{};
  int max_rows = 0, portion = 0, pool_pages = 0, pages_out = 0;
  int64_t next_id = 1;
  std::map<int64_t, std::unique_ptr<Request>> all;
  std::deque<Request*> waiting;
  std::vector<Request*> live;              // in order of admission
  std::vector<char> seq_used;
};

static void finish(cai_sched_s* s, Request* r)
{
  r->done = true;
  s->seq_used[r->seq] = 0; s->pages_out -= r->pages;
  (void)cai_decoder_reset(s->d, r->seq);
  r->seq = -1;
  s->live.erase(std::find(s->live.begin(), s->live.end(), r));
}

extern "C" int cai_sched_create(cai_decoder_t d, int max_rows, int portion, cai_sched_t* out)
{
  CAI_ENTER();
  CAI_REQUIRE(d && out, "cai_sched_create: null argument");
  cai_sched_s* s = new cai_sched_s();
  s->d = d;
  (void)cai_decoder_get_config(d, &s->cfg);
  s->max_rows = max_rows > 0 ? max_rows : 2048;
  s->portion = portion > 0 ? portion : 512;
  if (s->max_rows < s->cfg.max_batch) { delete s; return set_error(CAI_ERR_INVALID, "cai_sched_create: %d rows a step for %d sequences", max_rows, s->cfg.max_batch); }
  s->pool_pages = decoder_pool_pages(d);
  s->seq_used.assign((size_t)s->cfg.max_batch, 0);
  *out = s;
  return CAI_OK;
}

extern "C" int cai_sched_destroy(cai_sched_t s)
{
  CAI_ENTER();
  if (!s) return CAI_OK;
  while (!s->live.empty()) finish(s, s->live.back());
  delete s;
  return CAI_OK;
}

extern "C" int cai_sched_submit(cai_sched_t s, const int32_t* prompt, int n, int max_new, int eos, float temperature, int top_k, uint64_t seed, int64_t* id_out)
{
  CAI_ENTER();
  CAI_REQUIRE(s && prompt && id_out && n >= 1 && max_new >= 1, "cai_sched_submit: bad argument");
  CAI_REQUIRE(temperature <= 0.0f || (top_k >= 1 && top_k <= 1024), "cai_sched_submit: %d candidates (1..1024)", top_k);
  for (int i = 0; i < n; i++) CAI_REQUIRE(prompt[i] >= 0 && prompt[i] < s->cfg.vocab, "cai_sched_submit: token %d outside vocab %d", prompt[i], s->cfg.vocab);
  const int64_t total = (int64_t)n + max_new - 1;          // tokens that enter the cache: the last one drawn does not
  const int pages = decoder_peak_pages(s->d, total, s->portion);
  if (pages > s->pool_pages || (s->pool_pages == 0 && decoder_bounded(s->d) && total > s->cfg.max_ctx))
    return set_error(CAI_ERR_INVALID, "cai_sched_submit: %lld tokens do not fit the cache", (long long)total);
  auto r = std::make_unique<Request>();
  r->id = s->next_id++; r->prompt.assign(prompt, prompt + n); r->max_new = max_new; r->eos = eos;
  r->temperature = temperature; r->top_k = top_k; r->rng = seed; r->pages = pages;
  *id_out = r->id;
  s->waiting.push_back(r.get());
  s->all.emplace(r->id, std::move(r));
  return CAI_OK;
}

extern "C" int cai_sched_step(cai_sched_t s, int* live_out, int* waiting_out)
{
  CAI_ENTER();
  CAI_READY();
  CAI_REQUIRE(s, "cai_sched_step: null scheduler");
  // first come, first served: a request that does not fit yet holds back the ones behind it
  while (!s->waiting.empty()) {
    Request* r = s->waiting.front();
    const auto f = std::find(s->seq_used.begin(), s->seq_used.end(), 0);
    if (f == s->seq_used.end() || s->pages_out + r->pages > s->pool_pages) break;
    r->seq = (int)(f - s->seq_used.begin());
    *f = 1; s->pages_out += r->pages;
    (void)cai_decoder_reset(s->d, r->seq);
    s->live.push_back(r); s->waiting.pop_front();
  }
  if (!s->live.empty()) {
    std::vector<Request*> part = s->live;
    std::sort(part.begin(), part.end(), [](Request* a, Request* b) { return a->seq < b->seq; });
    int budget = s->max_rows;
    std::map<Request*, int> take;
    for (Request* r : s->live) if (r->fed == r->prompt.size()) { take[r] = 1; budget--; }
    for (Request* r : s->live) {
      if (r->fed == r->prompt.size() || budget <= 0) continue;
      const int m = std::min(std::min(s->portion, budget), (int)(r->prompt.size() - r->fed));
      take[r] = m; budget -= m;
    }
    std::vector<int32_t> seqs, counts, tokens;
    std::vector<uint8_t> want;
    std::vector<Request*> out;             // requests whose last row was wanted, in row order
    bool draws = false;
    for (Request* r : part) {
      const auto it = take.find(r);
      if (it == take.end()) continue;
      const int m = it->second;
      seqs.push_back(r->seq); counts.push_back(m);
      const bool prompt = r->fed < r->prompt.size();
      for (int i = 0; i < m; i++) tokens.push_back(prompt ? r->prompt[r->fed + i] : r->out.back());
      if (prompt) r->fed += m;
      want.insert(want.end(), (size_t)m, 0);
      if (r->fed == r->prompt.size()) { want.back() = 1; out.push_back(r); draws = draws || r->temperature > 0.0f; }
    }
    const bool on_device = decoder_keeps_rows(s->d);
    const int V = s->cfg.vocab;
    std::vector<int32_t> best(std::max<size_t>(out.size(), 1));
    std::vector<float> logits(draws && !on_device ? out.size() * (size_t)V : 0);
    int rc = cai_decoder_step_batch(s->d, (int)seqs.size(), seqs.data(), counts.data(), tokens.data(), want.data(), logits.empty() ? nullptr : logits.data(), best.data());
    if (rc) return rc;
    for (size_t k = 0; k < out.size(); k++) {
      Request* r = out[k];
      int32_t t = best[k];
      if (r->temperature > 0.0f) {
        std::vector<int32_t> tok((size_t)r->top_k); std::vector<float> p((size_t)r->top_k); int n = 0;
        rc = on_device ? cai_decoder_candidates(s->d, (int)k, nullptr, nullptr, 0, 1.0f, 0.0f, 0.0f, r->temperature, r->top_k, tok.data(), p.data(), &n)
                       : cai_sample_candidates(logits.data() + k * V, V, nullptr, nullptr, 0, 1.0f, 0.0f, 0.0f, r->temperature, r->top_k, tok.data(), p.data(), &n, 0);
        if (rc) return rc;
        double sum = 0.0, cum = 0.0; for (int i = 0; i < n; i++) sum += p[i];
        const double roll = r->draw() * sum;
        t = tok[std::max(n - 1, 0)];
        for (int i = 0; i < n; i++) { cum += p[i]; if (roll < cum) { t = tok[i]; break; } }
      }
      r->out.push_back(t);
      if ((int)r->out.size() >= r->max_new || t == r->eos) finish(s, r);
    }
  }
  if (live_out) *live_out = (int)s->live.size();
  if (waiting_out) *waiting_out = (int)s->waiting.size();
  return CAI_OK;
}

extern "C" int cai_sched_run(cai_sched_t s)
{
  CAI_ENTER();
  CAI_REQUIRE(s, "cai_sched_run: null scheduler");
  while (!s->live.empty() || !s->waiting.empty()) {
    const int rc = cai_sched_step(s, nullptr, nullptr);
    if (rc) return rc;
  }
  return CAI_OK;
}

extern "C" int cai_sched_result(cai_sched_t s, int64_t id, int32_t* tokens_out, int cap, int* n_out, int* done_out)
{
  CAI_ENTER();
  CAI_REQUIRE(s && n_out && (tokens_out || cap == 0), "cai_sched_result: null argument");
  const auto it = s->all.find(id);
  CAI_REQUIRE(it != s->all.end(), "cai_sched_result: no request %lld", (long long)id);
  const Request& r = *it->second;
  const int n = std::min((int)r.out.size(), cap);
  std::copy(r.out.begin(), r.out.begin() + n, tokens_out);
  *n_out = (int)r.out.size();
  if (done_out) *done_out = r.done;
  return CAI_OK;
}

extern "C" int cai_sched_drop(cai_sched_t s, int64_t id)
{
  CAI_ENTER();
  CAI_REQUIRE(s, "cai_sched_drop: null scheduler");
  const auto it = s->all.find(id);
  CAI_REQUIRE(it != s->all.end(), "cai_sched_drop: no request %lld", (long long)id);
  Request* r = it->second.get();
  if (r->seq >= 0) finish(s, r);
  else if (!r->done) s->waiting.erase(std::find(s->waiting.begin(), s->waiting.end(), r));
  s->all.erase(it);
  return CAI_OK;
}
