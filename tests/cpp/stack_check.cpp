// stack_check DIR N TOKENS... -- the C++ InferenceEngine on a model folder (config.json +
// model.safetensors): greedy continuation of a prompt, printed as "tokens: ...".
#include <cstdio>
#include <cstdlib>
#include <exception>
#include <vector>

#include "turboinfer/model/inference_engine.hpp"

int main(int argc, char** argv) {
  if (argc < 4) return 2;
  try {
    turboinfer::model::InferenceConfig cfg;
    cfg.max_sequence_length = 256;
    cfg.max_batch_size = 2;
    cfg.top_k = 1;
    turboinfer::model::InferenceEngine e(argv[1], cfg);
    std::vector<int> prompt;
    for (int i = 3; i < argc; ++i) prompt.push_back(std::atoi(argv[i]));
    const auto r = e.generate(prompt, (size_t)std::atoi(argv[2]));
    std::printf("%s\n%s\n", e.model_metadata().architecture.c_str(), e.performance_stats().c_str());
    std::printf("tokens:");
    for (int t : r.tokens) std::printf(" %d", t);
    std::printf("\n");
  } catch (const std::exception& ex) {
    std::fprintf(stderr, "%s\n", ex.what());
    return 1;
  }
  return 0;
}
