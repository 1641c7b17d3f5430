// Layer-stack models: decoders described by a list of layers, each with its own mixer and
// feed-forward.  A design registers a parser under its name (the `architecture` of its config.json)
// that turns the configuration into the mechanisms below; the pipeline, the cache and state managers and
// the loader work from that description and know no design by name.
#pragma once
#include <cstddef>
#include <cstdint>
#include <functional>
#include <map>
#include <memory>
#include <optional>
#include <string>
#include <vector>

#include "mini_json.h"
#include "nanoflow_kernels.h"

// Wavelengths above original / low are `factor` times longer, those below original / high as they are, and in between
// one goes over into the other.
struct RotationScaling {
  double factor = 1, low = 1, high = 4, original = 1;
};
struct RotationSpec {
  int dims = 0;
  double base = 1e4;
  bool interleaved = false;
  std::optional<RotationScaling> scaling = {};
  double frequency(int pair) const;
};

// q of position p is multiplied by 1 + coef * ln(floor((p + 1) / every) + 1).
struct QueryTemperatureSpec {
  double coef = 0;
  int every = 1;
};

// Softmax attention over a window with kept first positions; with `difference` the difference of two attentions per head over
// the same values, the second's weight being exp(lq1 . lk1) - exp(lq2 . lk2) + difference.
struct AttentionSpec {
  std::string prefix;  // of its tensors
  int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
  double scale = 1;
  int window = 0, keep_first = 0;  // window 0: everything before
  int chunk = 0;                   // positions see their own run of this many only, counted from 0; 0: all of one
  bool qk_norm = false;
  bool bias = false;       // of q, k and v
  bool sink = false;       // a score per head in the denominator, from a tensor
  bool unit_sink = false;  // the same with score 0
  bool head_gate = false;  // a head's output times the sigmoid of a projection of the input
  double softcap = 0;      // bound of the scores, 0: none
  int conv_taps = 0;       // short convolution of the projections over time, 0: none
  std::optional<double> difference;
  bool head_norm = false;  // a head's output divided by its root mean square
  int maps() const { return difference ? 2 : 1; }
  RotationSpec rot;
  bool value_norm = false;  // a value divided by its root mean square
  RotationSpec value_rot;   // of the values by their positions; a head's output is turned back by the query's
  std::optional<QueryTemperatureSpec> q_temp;
  double out_scale = 1;
};

// Softmax attention whose keys and values are projections of one cached latent row per position, plus a rotated
// key part that all heads share.
struct LatentAttentionSpec {
  std::string prefix;
  int heads = 0, dim = 0, rot_dim = 0, vdim = 0, kv_rank = 0;
  double scale = 1;
  int window = 0;    // 0: everything before
  RotationSpec rot;  // of the rotated part
};

// Linear recurrence with a state per head (nf_recurrence_kind).
struct RecurrenceSpec {
  std::string prefix;
  nf_recurrence_kind kind = NF_RECURRENCE_FIXED_DECAY;
  int heads = 0, dim = 0, vdim = 0;
  std::vector<double> decay;  // FIXED_DECAY
  RotationSpec rot;           // FIXED_DECAY
  double k_scale = 1;         // FIXED_DECAY
  nf_activation qkv_act = NF_ACT_NONE;  // FIXED_DECAY: of the projections
  // false: every head normed by itself, times silu(g); true: the concatenated heads normed together with a
  // weight, times sigmoid(g)
  bool joint_norm = false;
  double out_scale = 1;
};

struct MlpSpec {
  int ff = 0;
  nf_activation act = NF_ACT_SQUARED_RELU;
};
// Feed-forwards of which every token uses `top`; the router's last `identity` outputs stand for the input itself.  A token
// chooses from the keep_groups best of `groups` runs of outputs.  shared_ff > 0: one more feed-forward for every
// token, times the sigmoid of a projection.  It is held as always() experts of expertFf() columns beside the others, each
// a share of its columns: activations are taken column by column, so the shares' outputs add up to its own.
// With `gated` an expert has gate and up projections (nf_gated_act), each bounded by the expert's limit.
struct MixtureSpec {
  int experts = 0, identity = 0, top = 0, ff = 0;
  double scale = 1;
  nf_activation act = NF_ACT_GELU;
  int groups = 1, keep_groups = 1;
  bool correction = true;  // of the scores, where the choice is made
  nf_route_scores scores = NF_SCORES_SOFTMAX;
  bool weigh_input = false;  // a choice's weight multiplies the expert's input, not its output
  int shared_ff = 0;
  bool shared_gate = true;   // false: the shared feed-forward is added as it is
  struct Gated {
    double slope = 1, shift = 0, limit = 0, shared_limit = 0;
  };
  std::optional<Gated> gated;
  int outputs() const { return experts + identity; }
  int always() const {
    const int room = 64 - top < 1024 - experts ? 64 - top : 1024 - experts, shares = (shared_ff + ff - 1) / ff;
    return shared_ff > 0 ? (shares < room ? shares : room) : 0;
  }
  int expertFf() const { return shared_ff > 0 && (shared_ff + always() - 1) / always() > ff ? (shared_ff + always() - 1) / always() : ff; }
  int perToken() const { return top + always(); }
};
// A layer's mixer: attention, latent attention, a recurrence, or attention and a recurrence side by side on the same
// input; its feed-forward: dense, a mixture, or none.
struct LayerSpec {
  std::optional<AttentionSpec> attention;
  std::optional<LatentAttentionSpec> latent;
  std::optional<RecurrenceSpec> recurrence;
  std::optional<MlpSpec> mlp;
  std::optional<MixtureSpec> mixture;
  bool hasFeedForward() const { return mlp || mixture; }
};
// Layers [start, stop) run `times` times in a row, each pass with caches and states of its own.  Ahead of a pass its row of the
// tensor loop.step is added to the stream, and ahead of every pass but the first the embedding output as well.
struct LoopSpec {
  int start = 0, stop = 0, times = 1;
};
// One run of a layer; enters: the pass that starts with it, -1: none.
struct LayerRun {
  int layer = 0, enters = -1;
};

struct StackModelSpec {
  std::string architecture;
  int width = 0, vocab = 0;
  int max_positions = 0;  // 0: as many as the cache holds, up to 2^20
  double eps = 1e-5;
  bool learned_positions = false;
  nf_norm_kind norm = NF_NORM_RMS;  // of the residual stream (layer norms have a bias)
  bool pre_norm = false;            // x += f(norm(x)); else x += norm(f(x))
  bool post_norm = false;           // with pre_norm: x += normb(f(norm(x)))
  bool scalar_norms = false;        // the stream's norms have one weight for all columns
  bool layer_scale = false;         // what a sublayer adds is multiplied column by column, after its norm
  double embedding_scale = 1;
  double norm_offset = 0;           // added to the stored weights of the stream's norms
  double residual_scale = 1;        // of what a sublayer adds
  bool tied_head = false;           // the output projection is the embedding table
  double logit_scale = 1;
  int token_side = 0;               // size of the token input at the end of every layer, 0: none
  std::vector<LayerSpec> layers;
  std::optional<LoopSpec> loop;
  std::vector<LayerRun> runs() const;
  int ld() const { return (width + 7) / 8 * 8; }
  bool hasAttention() const {
    for (const auto& l : layers)
      if (l.attention) return true;
    return false;
  }
  bool hasState() const {
    for (const auto& l : layers)
      if (l.recurrence || (l.attention && l.attention->conv_taps > 1)) return true;
    return false;
  }
};

// ---- model registry
using StackParser = std::function<StackModelSpec(const mini_json::Value& config)>;
std::map<std::string, StackParser>& stackArchitectures();
struct RegisterStackArchitecture {
  RegisterStackArchitecture(const std::string& name, StackParser parser) { stackArchitectures()[name] = std::move(parser); }
};
// The description of a model configuration (its config.json); throws std::runtime_error with the reason when
// the architecture is unknown or the configuration is not complete.
StackModelSpec parseStackModel(const mini_json::Value& config);

// ---- named host tensors, and the safetensors file they come from
struct HostTensor {
  enum Type { BF16, F32, I32 } type = BF16;
  std::vector<int64_t> shape;
  const void* data = nullptr;
  size_t elements() const {
    size_t n = 1;
    for (int64_t d : shape) n *= (size_t)d;
    return n;
  }
};
using HostTensors = std::map<std::string, HostTensor>;

class SafetensorsFile {  // a read-only mapping; the tensors point into it
public:
  explicit SafetensorsFile(const std::string& path);
  ~SafetensorsFile();
  SafetensorsFile(const SafetensorsFile&) = delete;
  SafetensorsFile& operator=(const SafetensorsFile&) = delete;
  const HostTensors& tensors() const { return tensors_; }

private:
  void* map_ = nullptr;
  size_t bytes_ = 0;
  HostTensors tensors_;
};

// ---- device weights, in the form the operators take: projections that read the same input fused into
// one [N][K] matrix, N and K padded to 8 with zeros, vectors in fp32
struct DeviceMatrix {
  void* ptr = nullptr;
  int N = 0, K = 0;
};
struct AttentionWeights {
  DeviceMatrix qkv;  // and the heads' gate
  void* bias = nullptr;
  int q_col = 0, k_col = 0, v_col = 0, g_col = 0;
  float *q_norm = nullptr, *k_norm = nullptr, *sink = nullptr;
  void* conv = nullptr;  // [taps][columns of qkv]
  float map_weight = 0;
  nf_rotation rot{}, value_rot{};  // value_rot: pairs side by side, whatever the design's layout
};
struct LatentAttentionWeights {
  DeviceMatrix proj;  // q unrotated [heads][dim_pad] | q rotated [heads][rot_dim] | latent | rotated key part
  int q_col = 0, kv_col = 0;
  int dim_pad = 0, vdim_pad = 0;
  DeviceMatrix to_latent;    // per head [rank_pad][dim_pad]
  DeviceMatrix from_latent;  // per head [vdim_pad][rank_pad]
  DeviceMatrix expand;       // keys [heads][dim_pad], then (where from_latent is) values [heads][vdim_pad]
  float* norm = nullptr;
  nf_rotation rot{};
};
struct RecurrenceWeights {
  DeviceMatrix qkvg;                   // FIXED_DECAY; without g where the projections have an activation
  int q_col = 0, k_col = 0, v_col = 0, g_col = 0;
  float* log2_decay = nullptr;
  nf_rotation rot{};
  DeviceMatrix r, k, v, g, w1, w2;     // TOKEN_DECAY
  float *mu = nullptr, *w0 = nullptr, *u = nullptr, *norm = nullptr;  // mu [5][ld] in the order r k v g w
};
struct LayerWeights {
  AttentionWeights attention;
  LatentAttentionWeights latent;
  RecurrenceWeights recurrence;
  DeviceMatrix out;                    // over the attention heads, then the recurrence's
  DeviceMatrix up, down;               // of a mixture: per expert, one below the other
  DeviceMatrix router;
  float* correction = nullptr;
  nf_norm norm1{}, norm2{};            // pre_norm: of the sublayers' inputs
  nf_norm out_norm1{}, out_norm2{};    // of their outputs
  float* limits = nullptr;             // of a gated mixture's experts
  DeviceMatrix side_gate, side_proj;
  nf_norm side_norm{};
};
struct StackWeights {
  DeviceMatrix embed, pos, head, side_embed;
  float* loop_step = nullptr;  // [times][ld]
  nf_norm final_norm{};
  std::vector<LayerWeights> layers;
};

// What one pipeline serves: description, weights, caches and recurrent state, all on the device.
class StackModel {
public:
  // Uploads; throws std::runtime_error when a tensor is missing or has the wrong shape.
  StackModel(const StackModelSpec& spec, const HostTensors& tensors, nf_dtype dtype, int kv_pages, int page_size,
             int state_slots);
  ~StackModel();
  StackModel(const StackModel&) = delete;
  StackModel& operator=(const StackModel&) = delete;

  const StackModelSpec spec;
  const nf_dtype dtype;
  const int kv_pages, page_size, state_slots;
  const std::vector<LayerRun> runs;
  StackWeights weights;
  // per run of a layer; null where the layer has none
  std::vector<void*> kv_data;       // kv_pages pages (nf_kv_layout, nf_latent_layout)
  std::vector<float*> state;        // [state_slots][heads][dim_pad][vdim_pad]
  std::vector<float*> shift_state;  // [state_slots][ld]
  std::vector<void*> conv_state;    // [state_slots][taps - 1][columns of qkv]
  nf_kv_layout kvLayout(int layer) const;
  nf_latent_layout latentLayout(int layer) const;
  // of a latent layer's keys and values written out for all heads; page 0: heads too large for it, or fp32
  nf_kv_layout expandedLayout(int layer) const;
  size_t elementBytes() const { return dtype == NF_BF16 ? 2 : 4; }

private:
  struct Loader;
  std::vector<void*> owned_;
  std::map<std::vector<double>, float*> rotation_tables_;
  void* allocate(size_t bytes);  // zeroed device memory that lives as long as the model
  nf_rotation rotation(const RotationSpec& r);
};

// The model the current configuration names, and how it is to be held (set with the configuration).
struct StackModelConfig {
  StackModelSpec spec;
  nf_dtype dtype = NF_BF16;
  int kv_pages = 0, state_slots = 0;
};
extern std::shared_ptr<StackModelConfig> ActiveStackModel;  // null: a Llama-type model
