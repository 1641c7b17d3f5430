// Replays a trace: token ids given step by step on standard input, wanted logits to files.
//
//   trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N
//
// DIR of --model holds config.json and model.safetensors.  A line of standard input is one step,
//   {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["b"]}
// and is answered, once it has run, by a line "done <step>"; the wanted logits are in OUT/<step>.f32
// (little-endian fp32, [wanted][vocab]).  The cache pool holds N tokens, each request's rounded up to its pages;
// there are state slots for kSlots requests.
#include <cstdio>
#include <cstring>
#include <iostream>
#include <string>

#include "computeBound.h"
#include "config.h"
#include "mini_json.h"
#include "stackServe.h"

namespace {

constexpr int kSlots = 4;

int usage(const char* why) {
  std::fprintf(stderr, "trace_run: %s\nusage: trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N\n", why);
  return 2;
}

std::vector<int32_t> integers(const mini_json::Value& v) {
  std::vector<int32_t> out;
  for (const auto& x : v.arr) out.push_back((int32_t)x.number());
  return out;
}

std::string text_of(const mini_json::Value& v) {  // an id may be written as a number
  return v.kind == mini_json::Value::String ? v.str : std::to_string((long long)v.number());
}

void write_logits(const std::string& path, const std::vector<float>& v) {
  FILE* f = std::fopen(path.c_str(), "wb");
  if (!f) throw std::runtime_error("cannot write " + path);
  const size_t n = std::fwrite(v.data(), sizeof(float), v.size(), f);
  if (std::fclose(f) != 0 || n != v.size()) throw std::runtime_error("cannot write " + path);
}

}  // namespace

int main(int argc, char** argv) {
  std::string model, dtype, out;
  long max_tokens = 0;
  for (int i = 1; i < argc; ++i) {
    const std::string a = argv[i];
    if (i + 1 >= argc) return usage((a + " needs a value").c_str());
    const char* v = argv[++i];
    if (a == "--model") model = v;
    else if (a == "--dtype") dtype = v;
    else if (a == "--out") out = v;
    else if (a == "--max-tokens") max_tokens = std::strtol(v, nullptr, 10);
    else return usage(("unknown option " + a).c_str());
  }
  if (model.empty() || out.empty() || max_tokens <= 0) return usage("--model, --out and --max-tokens are required");
  if (dtype != "bfloat16" && dtype != "float32") return usage("--dtype is bfloat16 or float32");
  try {
    const int page = 16;
    const int pages = (int)((max_tokens + page - 1) / page);
    std::string error;
    if (!setStackModelConfig(mini_json::parse_file(model + "/config.json"), dtype, (int)max_tokens, pages, kSlots, &error))
      throw std::runtime_error(model + "/config.json: " + error);
    {
      const SafetensorsFile file(model + "/model.safetensors");
      startStackPipeline(file.tensors(), (int)max_tokens);
    }
    StackReplay replay(pages, page, kSlots);
    std::string line;
    while (std::getline(std::cin, line)) {
      if (line.find_first_not_of(" \t\r") == std::string::npos) continue;
      const mini_json::Value j = mini_json::Parser(line).parse();
      const std::string step = text_of(j.at("step"));
      std::vector<StackReplay::Entry> entries;
      if (j.contains("entries"))
        for (const auto& e : j.at("entries").arr)
          entries.push_back({text_of(e.at("id")), integers(e.at("tokens")), e.contains("want") ? integers(e.at("want")) : std::vector<int32_t>()});
      const std::vector<float> logits = replay.step(entries);
      if (!logits.empty()) write_logits(out + "/" + step + ".f32", logits);
      if (j.contains("end"))
        for (const auto& id : j.at("end").arr) replay.end(text_of(id));
      std::printf("done %s\n", step.c_str());
      std::fflush(stdout);
    }
    finalize();
    return 0;
  } catch (const std::exception& e) {
    std::fprintf(stderr, "trace_run: %s\n", e.what());
    finalize();
    return 1;
  }
}
