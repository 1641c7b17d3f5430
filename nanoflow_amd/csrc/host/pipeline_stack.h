// LayerStackPipeline: one iteration of a layer-stack model (stackModel.h) behind PipelineBase's
// config / update / run.  Decode rows first, then the portions of prompts, as in the other schedules;
// the two mixers of a layer that has both run on two streams.
#pragma once
#include "pipeline.h"
#include "stackOperators.h"

class LayerStackPipeline : public PipelineBase {
public:
  LayerStackPipeline(vortexInitData* input_data, int nrank, int nranks, int vnranks);
  ~LayerStackPipeline() override;
  vortexOutputData run() override;
  void update(vortexUpdateData* update_data) override;
  void config(vortexConfigData* config_data) override;
  void setName() override;
  void setProfiling(int level) override;
  hipStream_t uploadStream() override { return stream_all; }

  // Bytes of tmp buffer that a batch of max_rows rows takes.
  static size_t tmpBytes(const StackModel& model, int max_rows);
  // Rows of logits one iteration can compute.
  static int maxLogitRows(const StackModelSpec& spec, int max_rows);

  // fp32 logits of the last iteration: [logitRows()][vocab], row stride logitLd() (device memory).
  const float* logits() const { return buf.logits; }
  int logitRows() const { return batch.logit_rows; }
  int logitLd() const { return model->weights.head.N; }
  int vocab() const { return model->spec.vocab; }
  // The residual stream [rows][ld]; with keepLayers(true) before config(), also after every layer
  // run of a layer ([runs][max rows][ld]; eager iterations only).
  const float* residual() const { return buf.x; }
  const float* layerOutputs() const { return layer_outputs; }
  int rows() const { return batch.rows; }
  int maxRows() const { return config_data.global_batch_size; }
  static inline bool keep_layers = false;

private:
  struct Buffers {
    float* x = nullptr;        // residual stream
    void* act = nullptr;       // what the next sublayer reads: x, normed or as it is (then x itself in fp32)
    void* attn_proj = nullptr; // q | k | v rows
    void* q = nullptr;         // normed, rotated queries
    void* mix = nullptr;       // token-shifted inputs [5][rows][ld], also q | k | v | g rows of a fixed-decay layer
    void* rkvg[4] = {};
    float* w1_sums = nullptr;
    void* w1_act = nullptr;
    float* z = nullptr;
    void* heads = nullptr;     // the mixers' heads, side by side
    void* latent = nullptr;    // [rows][heads][rank_pad]
    void *latent_q = nullptr, *latent_rows = nullptr, *latent_products = nullptr, *latent_pages = nullptr;  // the prompts' keys and values, written out
    int32_t* latent_page_ids = nullptr;
    int latent_max_pages = 0;
    nf_routing routing{};
    float *router_sums = nullptr, *side_sums = nullptr;
    void *expert_ff = nullptr, *expert_out = nullptr;  // sorted rows
    void* side = nullptr;
    void* y = nullptr;         // a sublayer's output in the activations' type
    float* y_sums = nullptr;   // ... or as fp32 sums
    void* ff = nullptr;
    void* head_in = nullptr;
    float* logits = nullptr;
    int32_t* argmax = nullptr;
    void *gemm_ws = nullptr, *gemm_ws_side = nullptr, *recur_ws = nullptr, *latent_ws = nullptr;
    size_t y_sums_bytes = 0, w1_sums_bytes = 0, z_bytes = 0, logits_bytes = 0, gemm_ws_bytes = 0, recur_ws_bytes = 0, latent_ws_bytes = 0,
           router_sums_bytes = 0, side_sums_bytes = 0;
  };
  static Buffers plan(const StackModel& m, int T, AllocationManager<half>& arena);
  void enqueueIteration();
  // run: of a layer, in the model's order of runs
  void enqueueMixer(int run);
  // What the row operator at the end of a sublayer leaves for the next one.
  struct Next {
    bool wanted = false;
    nf_norm norm{};   // NF_NORM_NONE: x as it is
    int enters = -1;  // the pass over looped layers that it starts
  };
  Next beforeRun(int run) const;
  Next afterMixer(int run) const;
  Next afterFeedForward(int run) const;
  Next afterLayer(int run) const;
  void enterRun(int run);
  void setNext(const Next& next);
  // the residual stream as a sublayer reads it without a norm
  const void* plain() const { return model->dtype == NF_BF16 ? buf.act : buf.x; }
  const void* sublayerInput() const { return model->spec.pre_norm ? buf.act : plain(); }
  void sublayerOut(const void* a, const DeviceMatrix& w, const nf_norm& y_norm, const Next& next);
  void mixtureOut(int run);
  void tokenSide(int run);
  int expandPages(int layer) const;
  void latentBranch(int run);
  void attentionBranch(int run, hipStream_t s);
  void recurrenceBranch(int run);

  StackModel* model;
  Buffers buf;
  StackBatch batch;
  StackEmbedding embedding;
  StackLinear linear, linear_side;
  StackNorm firstNorm;
  StackResidual residualAdd;
  StackGroupedLinear grouped;
  StackRouter router;
  StackTokenGate tokenGate;
  StackGatedNorm gatedNorm;
  StackLatentAppend latentAppend;
  StackLatentAttention latentAttention;
  StackLatentExpand latentExpand;
  StackLatentQueries latentQueries;
  StackTokenShift tokenShift;
  StackTanh tanhRows;
  StackQKVAppend qkvAppend;
  StackAttention attention;
  StackRecurrence recurrence;
  StackGatherNorm gatherNorm;
  StackArgmax sampler;
  float* layer_outputs = nullptr;
  vortexOutputData output_data;
  hipStream_t stream_all = nullptr, stream_side = nullptr;
  hipEvent_t fork = nullptr, join = nullptr;
};
