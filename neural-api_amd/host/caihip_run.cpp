// Command-line twin of the reference's greedy decode loop (TChatEngine.GenerateFromIds,
// neural/neuralchatengine.pas:1428-1561, greedy branch 1493-1494; --stats timing 1590-1605) over token ids:
//   caihip_run MODEL N_NEW [--max-ctx N] [--stepwise] [--dtype bfloat16|float32] TOKEN_ID...
//   caihip_run MODEL N_NEW --batch [--sequences S] [--portion P] [--temperature T --top-k K --seed N] TOKEN_ID... [-- TOKEN_ID...]...
// MODEL is a GGUF file or a folder with config.json and model.safetensors.  Prefills the prompt, then decodes N_NEW tokens
// greedily and prints them on one line; a second line reports the prompt and decode rates the way --stats does (tokens /
// (t_end - t_first)).  With --batch every prompt (they are separated by --) is a request of the continuous-batching scheduler
// and prints a line of its own, in the order given.  Tokenisation stays with the caller.
#include "caihip_host.hpp"

#include <chrono>
#include <cstdlib>
#include <cstring>
#include <memory>
#include <sys/stat.h>

int main(int argc, char** argv)
{
  if (argc < 4) { std::fprintf(stderr, "usage: %s MODEL N_NEW [--max-ctx N] [--stepwise] [--dtype bfloat16|float32] [--batch] [--sequences S] [--portion P] [--temperature T] [--top-k K] [--seed N] TOKEN_ID... [-- TOKEN_ID...]\n", argv[0]); return 2; }
  const std::string model = argv[1];
  const int n_new = std::atoi(argv[2]);
  int max_ctx = 0, dtype = CAI_DTYPE_BF16, sequences = 4, portion = 0, top_k = 40; bool stepwise = false, batch = false;
  float temperature = 0.0f; unsigned long long seed = 0;
  std::vector<std::vector<int32_t>> prompts(1);
  for (int i = 3; i < argc; i++) {
    if (!std::strcmp(argv[i], "--max-ctx") && i + 1 < argc) max_ctx = std::atoi(argv[++i]);
    else if (!std::strcmp(argv[i], "--stepwise")) stepwise = true;
    else if (!std::strcmp(argv[i], "--batch")) batch = true;
    else if (!std::strcmp(argv[i], "--sequences") && i + 1 < argc) sequences = std::atoi(argv[++i]);
    else if (!std::strcmp(argv[i], "--portion") && i + 1 < argc) portion = std::atoi(argv[++i]);
    else if (!std::strcmp(argv[i], "--temperature") && i + 1 < argc) temperature = (float)std::atof(argv[++i]);
    else if (!std::strcmp(argv[i], "--top-k") && i + 1 < argc) top_k = std::atoi(argv[++i]);
    else if (!std::strcmp(argv[i], "--seed") && i + 1 < argc) seed = std::strtoull(argv[++i], nullptr, 10);
    else if (!std::strcmp(argv[i], "--dtype") && i + 1 < argc) dtype = !std::strcmp(argv[++i], "float32") ? CAI_DTYPE_F32 : CAI_DTYPE_BF16;
    else if (!std::strcmp(argv[i], "--")) prompts.emplace_back();
    else prompts.back().push_back((int32_t)std::atoi(argv[i]));
  }
  const std::vector<int32_t>& prompt = prompts[0];
  for (auto& p : prompts) if (p.empty()) { std::fprintf(stderr, "an empty prompt\n"); return 2; }
  if (prompts.size() > 1) batch = true;
  struct stat sb;
  const bool folder = stat(model.c_str(), &sb) == 0 && S_ISDIR(sb.st_mode);
  if (prompt.empty() || n_new < 1) { std::fprintf(stderr, "need at least one prompt token and N_NEW >= 1\n"); return 2; }
  try {
    caihip::EnableHIP(0);
    if (batch) {
      size_t need = 0;
      for (auto& p : prompts) need = std::max(need, p.size() + (size_t)n_new);
      sequences = std::min(std::max(sequences, 1), 8);
      caihip::TNNetStreamingDecoder dec(model, max_ctx > 0 ? max_ctx : (int)((need + 63) / 64 * 64) * (folder ? sequences : 1), sequences, dtype);
      caihip::TBatchScheduler sched(dec, 0, portion);
      std::vector<int64_t> ids;
      for (auto& p : prompts) ids.push_back(sched.Submit(p, n_new, -1, temperature, top_k, seed + ids.size()));
      sched.Run();
      for (int64_t id : ids) {
        const std::vector<int32_t> out = sched.Result(id);
        for (size_t i = 0; i < out.size(); i++) std::printf("%s%d", i ? " " : "", out[i]);
        std::printf("\n");
      }
      return 0;
    }
    std::unique_ptr<caihip::TNNetStreamingDecoder> holder(folder
      ? new caihip::TNNetStreamingDecoder(model, max_ctx > 0 ? max_ctx : (int)prompt.size() + n_new, 1, dtype)
      : new caihip::TNNetStreamingDecoder(model, max_ctx));
    caihip::TNNetStreamingDecoder& dec = *holder;
    using clk = std::chrono::steady_clock;
    const auto t0 = clk::now();
    dec.Reset();
    if (stepwise) for (size_t i = 0; i < prompt.size(); i++) dec.StepForward(&prompt[i], 1, (int)i);
    else dec.StepForward(prompt.data(), (int)prompt.size(), 0);
    const auto t1 = clk::now();
    std::vector<int32_t> out;
    out.push_back(dec.ArgMaxRow());
    if (n_new > 1) {
      if (stepwise) {
        for (int k = 1; k < n_new; k++) { const int32_t t = out.back(); dec.StepForward(&t, 1, (int)prompt.size() + k - 1); out.push_back(dec.ArgMaxRow()); }
      } else {
        const std::vector<int32_t> more = dec.GenerateGreedy(out[0], (int)prompt.size(), n_new - 1);
        out.insert(out.end(), more.begin(), more.end());
      }
    }
    const auto t2 = clk::now();
    for (size_t i = 0; i < out.size(); i++) std::printf("%s%d", i ? " " : "", out[i]);
    std::printf("\n");
    const double tp = std::chrono::duration<double>(t1 - t0).count(), td = std::chrono::duration<double>(t2 - t1).count();
    std::printf("stats: prompt %zu tok %.1f tok/s, decode %d tok %.1f tok/s, cache %d\n", prompt.size(), prompt.size() / (tp > 0 ? tp : 1e-9),
                n_new - 1, (n_new - 1) / (td > 0 ? td : 1e-9), dec.SDPACacheLength());
  } catch (const caihip::CaiError& e) {
    std::fprintf(stderr, "caihip_run: error %d: %s\n", e.code, e.what());
    return 1;
  }
  return 0;
}
