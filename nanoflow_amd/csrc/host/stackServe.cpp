#include "stackServe.h"

#include <algorithm>
#include <stdexcept>

#include "computeBound.h"
#include "pipeline_stack.h"

void startStackPipeline(const HostTensors& tensors, int global_batch) {
  if (!ActiveStackModel) throw std::runtime_error("no layer-stack model is configured");
  if (currentPipeline()) throw std::runtime_error("a pipeline is running already");
  const StackModelConfig& c = *ActiveStackModel;
  HIP_CHECK(hipSetDevice(0));
  std::vector<vortexInitData> in(1);
  in[0].stack = std::make_shared<StackModel>(c.spec, tensors, c.dtype, c.kv_pages, ModelConfig.frame_page_size, c.state_slots);
  in[0].tmp_buffer_size = (LayerStackPipeline::tmpBytes(*in[0].stack, global_batch) + 1) / 2;
  HIP_CHECK(hipMalloc(&in[0].tmp_buffer, in[0].tmp_buffer_size * sizeof(half)));
  // the buffer is freed with the model, after the pipeline that plans into it
  in[0].stack = std::shared_ptr<StackModel>(in[0].stack.get(), [model = in[0].stack, tmp = in[0].tmp_buffer](StackModel*) mutable {
    (void)hipFree(tmp);
    model.reset();
  });
  static std::vector<vortexOutputData> outputs_of_worker(1);  // the worker keeps a pointer to it
  init(1, 1, in, outputs_of_worker, Worker::PipelineType::LAYER_STACK);
  static std::vector<vortexConfigData> cfg(1);
  cfg[0] = vortexConfigData();
  cfg[0].global_batch_size = global_batch;
  config(1, cfg);
  if (PipelineBase* p = currentPipeline(); p && !p->configError().empty()) {
    const std::string e = p->configError();
    finalize();
    throw std::runtime_error(e);
  }
}

StackReplay::StackReplay(int kv_pages, int page_size, int state_slots) : pool_(kv_pages, page_size), states_(state_slots) {}

void StackReplay::end(const std::string& id) {
  auto it = requests_.find(id);
  if (it == requests_.end()) return;
  it->second->release();
  requests_.erase(it);
}

std::vector<float> StackReplay::step(const std::vector<Entry>& entries) {
  auto* pipeline = dynamic_cast<LayerStackPipeline*>(currentPipeline());
  if (!pipeline) throw std::runtime_error("no layer-stack pipeline is running");
  const StackModelSpec& spec = ActiveStackModel->spec;
  // single tokens of requests that have started are decode rows, everything else is a portion
  std::vector<size_t> order;
  size_t n_decode = 0;
  for (int pass = 0; pass < 2; ++pass)
    for (size_t i = 0; i < entries.size(); ++i) {
      if (entries[i].tokens.empty()) throw std::runtime_error("request " + entries[i].id + " brings no tokens");
      auto it = requests_.find(entries[i].id);
      const bool decode = entries[i].tokens.size() == 1 && it != requests_.end() && it->second->seqlen() > 0;
      if (decode == (pass == 0)) order.push_back(i);
      if (pass == 0 && decode) ++n_decode;
    }
  std::vector<BatchEntry> decode, prefill;
  std::vector<int32_t> decode_tokens, wanted;
  FormedBatch b;
  std::vector<int> first_row(entries.size(), 0);
  int rows = 0;
  for (size_t k = 0; k < order.size(); ++k) {
    const Entry& e = entries[order[k]];
    auto& cache = requests_[e.id];
    if (!cache) cache = std::make_unique<KVCache>(&pool_, &states_);
    if (cache->seqlen() + (int)e.tokens.size() > spec.max_positions)
      throw std::runtime_error("request " + e.id + " is longer than the model's " + std::to_string(spec.max_positions) + " positions");
    for (int32_t t : e.tokens)
      if (t < 0 || t >= spec.vocab) throw std::runtime_error("token " + std::to_string(t) + " is beyond the vocabulary");
    for (const BatchEntry& other : k < n_decode ? decode : prefill)
      if (other.cache == cache.get()) throw std::runtime_error("request " + e.id + " appears twice in a step");
    cache->allocate_tokens((int)e.tokens.size());
    first_row[order[k]] = rows;
    rows += (int)e.tokens.size();
    if (k < n_decode) {
      decode.push_back({1, cache.get()});
      decode_tokens.push_back(e.tokens[0]);
    } else {
      prefill.push_back({(int)e.tokens.size(), cache.get()});
      b.input_tokens.insert(b.input_tokens.end(), e.tokens.begin(), e.tokens.end());
    }
  }
  for (size_t i = 0; i < entries.size(); ++i)
    for (int32_t w : entries[i].want) {
      if (w < 0 || w >= (int)entries[i].tokens.size()) throw std::runtime_error("request " + entries[i].id + " wants a place it does not bring");
      wanted.push_back(first_row[i] + w);
    }
  if (rows == 0) return {};
  if (rows > pipeline->maxRows()) throw std::runtime_error("a step of " + std::to_string(rows) + " tokens exceeds the batch size");
  if ((int)wanted.size() > LayerStackPipeline::maxLogitRows(spec, pipeline->maxRows()))
    throw std::runtime_error("a step wants the logits of " + std::to_string(wanted.size()) + " tokens");
  assembleBatch(decode, prefill, b);

  static std::vector<vortexUpdateData> upd(1);
  vortexUpdateData& u = upd[0];
  u = vortexUpdateData();
  u.decodePrefillBorder = (int)decode.size();
  u.prefillNum = (int)prefill.size();
  u.prefillTokensNum = (int)b.input_tokens.size();
  u.input_tokens = b.input_tokens.data();
  u.input_indptr = b.input_indptr.data();
  u.rev_input_indptr = b.rev_input_indptr.data();
  u.kv_indptr = b.kv_indptr.data();
  u.kv_indices = b.kv_indices.data();
  u.kv_last_page_len = b.kv_last_page_len.data();
  u.per_token_offset = b.per_token_offset.data();
  int32_t groups[4] = {(int32_t)decode.size(), 0, 0, 0}, blocks[4] = {0, 0, 0, 0};
  u.gemv_batch_size = groups;
  u.gemv_num_blocks = blocks;
  u.state_slots = b.state_slots.data();
  static int32_t none = 0;
  u.logit_rows = wanted.empty() ? &none : wanted.data();
  u.logit_rows_num = (int)wanted.size();
  if (decode_tokens.empty()) decode_tokens.push_back(0);
  u.decode_tokens = decode_tokens.data();
  update(1, upd);
  run();

  std::vector<float> logits(wanted.size() * (size_t)spec.vocab);
  if (!logits.empty())
    HIP_CHECK(hipMemcpy2D(logits.data(), (size_t)spec.vocab * 4, pipeline->logits(), (size_t)pipeline->logitLd() * 4,
                          (size_t)spec.vocab * 4, wanted.size(), hipMemcpyDeviceToHost));
  return logits;
}
