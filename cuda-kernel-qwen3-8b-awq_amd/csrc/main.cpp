// Command-line harness with the behaviour of the reference's main
// (Inference.cu:1413-1433): one argument, BOS prompt, 20 greedy tokens.
// Options behind the folder choose another prompt, length or number format; the
// folder may be of any model class (awq_open).
#include <cstdlib>
#include <iostream>
#include <sstream>
#include <string>
#include <vector>

#include "../../include/awq_infer.h"
#include "qwen3_awq_infer.hpp"

static int usage(const char* program) {
  std::cerr << "Usage: " << program << " <path_to_weight_folder> [--prompt id,id,...] [--new n] [--dtype bfloat16|float32]"
            << " [--max-positions n]\n";
  return 1;
}

int main(int argc, char** argv) {
  if (argc < 2) return usage(argv[0]);
  std::string weight_dir = argv[1];
  std::vector<int> prompt = {151643};
  int max_new_tokens = 20;
  awq_open_options options{};
  for (int i = 2; i < argc; i += 2) {
    if (i + 1 >= argc) return usage(argv[0]);
    const std::string key = argv[i], value = argv[i + 1];
    if (key == "--prompt") {
      prompt.clear();
      std::stringstream s(value);
      for (std::string id; std::getline(s, id, ',');) prompt.push_back(std::atoi(id.c_str()));
    } else if (key == "--new") {
      max_new_tokens = std::atoi(value.c_str());
    } else if (key == "--dtype" && value == "bfloat16") {
      options.dtype = AWQ_DTYPE_BFLOAT16;
    } else if (key == "--dtype" && value == "float32") {
      options.dtype = AWQ_DTYPE_FLOAT32;
    } else if (key == "--max-positions") {
      options.max_positions = std::atoll(value.c_str());
    } else {
      return usage(argv[0]);
    }
  }
  QWen3AWQInfer infer(weight_dir, options);

  std::vector<int> out = infer.generateResponse(prompt, max_new_tokens);

  std::cout << "Generated tokens: ";
  for (int tok : out) std::cout << tok << " ";
  std::cout << std::endl;
  return 0;
}
