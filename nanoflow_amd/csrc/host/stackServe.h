// Set-up of a layer-stack pipeline, and the replay of given tokens through it.
#pragma once
#include <map>
#include <memory>
#include <string>
#include <vector>

#include "batchFormer.h"
#include "stackModel.h"

// Loads the model the configuration names (setStackModelConfig) from named host tensors, allocates the
// schedule's buffers for global_batch rows and starts the pipeline.  Throws std::runtime_error.
void startStackPipeline(const HostTensors& tensors, int global_batch);

// Feeds given token ids through the pipeline step by step: every step is one iteration of the
// schedule that serves the model, its batch put together from the same page pool, state slots and
// batch assembly as the batch former's.
class StackReplay {
public:
  struct Entry {
    std::string id;
    std::vector<int32_t> tokens;
    std::vector<int32_t> want;  // places among the tokens whose logits are wanted
  };
  StackReplay(int kv_pages, int page_size, int state_slots);
  // Logits [wanted][vocab] in the order of the entries and of their wants.  Throws std::runtime_error (a token
  // beyond the vocabulary, a request beyond the positions, no page or slot left); the replay is then over.
  std::vector<float> step(const std::vector<Entry>& entries);
  void end(const std::string& id);
  int live() const { return (int)requests_.size(); }
  int free_pages() const { return pool_.num_free_pages(); }
  int free_slots() const { return states_.num_free(); }

private:
  KVPool pool_;
  StatePool states_;
  std::map<std::string, std::unique_ptr<KVCache>> requests_;
};
