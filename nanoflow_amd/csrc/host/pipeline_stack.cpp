#include "pipeline_stack.h"

#include <algorithm>

#include "pipelineFactory.h"

namespace {

// A projection back to the residual width that is not split over K is rounded before the norm reads it
// when it has more than this many rows (fp32 rows would cost more than they are worth there); otherwise the
// norm adds the fp32 shares itself.
constexpr int kSumsMaxRows = 512;
constexpr int kSumsMaxShares = 16;
// The prompts of an iteration have their keys and values written out of the latents for contexts of at most this many
// tokens together (or twice the iteration's rows), rounded up to whole groups of pages.
constexpr int kExpandTokens = 8192, kExpandGroup = 64;

const RegisterPipeline registered(Worker::PipelineType::LAYER_STACK, [](vortexInitData* input, int rank, int nranks, int vnranks) {
  return std::unique_ptr<PipelineBase>(new LayerStackPipeline(input, rank, nranks, vnranks));
});

}  // namespace

LayerStackPipeline::LayerStackPipeline(vortexInitData* input_data, int nrank, int nranks, int vnranks)
    : PipelineBase(input_data, nrank, nranks, vnranks), model(input_data->stack.get()) {
  stream_all = createPipelineStream(0, 0);
  stream_side = createPipelineStream(0, 0);
  HIP_CHECK(hipEventCreateWithFlags(&fork, hipEventDisableTiming));
  HIP_CHECK(hipEventCreateWithFlags(&join, hipEventDisableTiming));
}

LayerStackPipeline::~LayerStackPipeline() {
  clearGraphs();
  delete[] output_data.sampled_token_array;
  if (layer_outputs) (void)hipFree(layer_outputs);
  if (fork) (void)hipEventDestroy(fork);
  if (join) (void)hipEventDestroy(join);
  if (stream_side) (void)hipStreamDestroy(stream_side);
  if (stream_all) (void)hipStreamDestroy(stream_all);
}

int LayerStackPipeline::maxLogitRows(const StackModelSpec& spec, int max_rows) {
  const size_t fit = ((size_t)1 << 30) / (4 * (size_t)((spec.vocab + 7) / 8 * 8));  // 1 GiB of logits
  return (int)std::min<size_t>((size_t)max_rows, std::max<size_t>(fit, 1));
}

LayerStackPipeline::Buffers LayerStackPipeline::plan(const StackModel& m, int T, AllocationManager<half>& arena) {
  const StackModelSpec& spec = m.spec;
  const size_t es = m.elementBytes(), ld = (size_t)spec.ld();
  const bool bf16 = m.dtype == NF_BF16;
  Buffers b;
  size_t attn_proj = 0, q = 0, mix = 0, rk = 0, vg = 0, w1 = 0, z = 0, heads = 0, ff = 0, ws = 0, ws_side = 0, recur = 0;
  size_t expand_n = 0, latent_q = 0, expand_rank = 0, expand_page = 0, latent = 0, top = 0, experts = 0, expert_ff = 0, tiles = 0, side = 0;
  auto few = [&](const DeviceMatrix& w) { return bf16 ? nf_gemm_nk_workspace_bytes_upto(T, w.N, w.K) : 0; };
  auto sums = [&](int rows, const DeviceMatrix& w, int shares) {
    return bf16 ? nf_gemm_nk_sums_bytes_upto(rows, w.N, w.K, shares) : (size_t)rows * w.N * 4;
  };
  for (size_t i = 0; i < spec.layers.size(); ++i) {
    const LayerSpec& s = spec.layers[i];
    const LayerWeights& w = m.weights.layers[i];
    if (s.attention) {
      attn_proj = std::max(attn_proj, (size_t)w.attention.qkv.N);
      q = std::max(q, (size_t)s.attention->heads * s.attention->maps() * m.kvLayout((int)i).k_pad);
      ws_side = std::max(ws_side, few(w.attention.qkv));
    }
    if (s.recurrence) {
      const RecurrenceSpec& r = *s.recurrence;
      recur = std::max(recur, nf_recurrence_workspace_bytes(r.heads, r.dim, r.vdim, T, T));
      if (r.kind == NF_RECURRENCE_FIXED_DECAY) {
        mix = std::max(mix, (size_t)w.recurrence.qkvg.N);
        ws = std::max(ws, few(w.recurrence.qkvg));
        if (w.recurrence.g.N > 0) {
          vg = std::max(vg, (size_t)w.recurrence.g.N);
          ws = std::max(ws, few(w.recurrence.g));
        }
      } else {
        mix = std::max(mix, 5 * ld);
        rk = std::max(rk, (size_t)w.recurrence.r.N);
        vg = std::max(vg, (size_t)w.recurrence.v.N);
        w1 = std::max(w1, (size_t)w.recurrence.w1.N);
        z = std::max(z, (size_t)w.recurrence.w2.N);
        b.w1_sums_bytes = std::max(b.w1_sums_bytes, sums(T, w.recurrence.w1, kSumsMaxShares));
        b.z_bytes = std::max(b.z_bytes, sums(T, w.recurrence.w2, 1));
        ws = std::max({ws, few(w.recurrence.r), few(w.recurrence.v)});
      }
    }
    if (s.latent) {
      const nf_latent_layout l = m.latentLayout((int)i);
      attn_proj = std::max(attn_proj, (size_t)w.latent.proj.N);
      q = std::max(q, (size_t)l.heads * l.row_ld);
      latent = std::max(latent, (size_t)l.heads * l.rank_pad);
      ws = std::max(ws, few(w.latent.proj));
      if (const nf_kv_layout x = m.expandedLayout((int)i); x.page > 0) {
        latent_q = std::max(latent_q, (size_t)x.heads * x.k_pad);
        expand_n = std::max(expand_n, (size_t)w.latent.expand.N);
        expand_rank = std::max(expand_rank, (size_t)l.rank_pad);
        expand_page = std::max(expand_page, nf_kv_page_elements(&x));
        ws = std::max(ws, few(w.latent.expand));
      }
      b.latent_ws_bytes = std::max(b.latent_ws_bytes, nf_latent_workspace_bytes(&l, T));
    }
    if (s.mixture) {
      const MixtureSpec& x = *s.mixture;
      top = std::max(top, (size_t)x.perToken());
      experts = std::max(experts, (size_t)(x.experts + x.always()));
      expert_ff = std::max(expert_ff, (size_t)x.perToken() * w.down.K);
      tiles = std::max(tiles, (size_t)nf_routing_max_tiles(T * x.perToken(), x.experts + x.always(), 64));
      b.router_sums_bytes = std::max(b.router_sums_bytes, sums(T, w.router, kSumsMaxShares));
    }
    if (spec.token_side > 0) {
      side = std::max(side, (size_t)w.side_gate.N);
      b.side_sums_bytes = std::max(b.side_sums_bytes, sums(T, w.side_gate, kSumsMaxShares));
      b.y_sums_bytes = std::max(b.y_sums_bytes, sums(T, w.side_proj, kSumsMaxShares));
    }
    heads = std::max(heads, (size_t)w.out.K);
    b.y_sums_bytes = std::max(b.y_sums_bytes, sums(T, w.out, kSumsMaxShares));
    if (s.mlp) {
      ff = std::max(ff, (size_t)w.up.N);
      ws = std::max(ws, few(w.up));
      b.y_sums_bytes = std::max(b.y_sums_bytes, sums(T, w.down, kSumsMaxShares));
    }
  }
  const int L = maxLogitRows(spec, T);
  b.logits_bytes = sums(L, m.weights.head, 1);
  b.gemm_ws_bytes = std::max(ws, ws_side);
  b.recur_ws_bytes = recur;
  b.x = (float*)arena.allocBytes(T * ld * 4);
  b.act = bf16 || spec.pre_norm ? arena.allocBytes(T * ld * es) : b.x;
  b.attn_proj = arena.allocBytes(T * attn_proj * es);
  b.q = arena.allocBytes(T * q * es);
  b.mix = arena.allocBytes(T * mix * es);
  for (int i = 0; i < 4; ++i) b.rkvg[i] = arena.allocBytes(T * (i < 2 ? rk : vg) * es);
  b.w1_sums = (float*)arena.allocBytes(b.w1_sums_bytes);
  b.w1_act = arena.allocBytes(T * w1 * es);
  b.z = (float*)arena.allocBytes(std::max(b.z_bytes, T * z * 4));
  b.heads = arena.allocBytes(T * heads * es);
  b.latent = arena.allocBytes(T * latent * es);
  if (expand_n > 0) {
    const int pages = std::min(m.kv_pages, std::max(2 * T, kExpandTokens) / m.page_size);
    b.latent_max_pages = (pages + kExpandGroup - 1) / kExpandGroup * kExpandGroup;
    const size_t rows = (size_t)b.latent_max_pages * m.page_size;
    b.latent_q = arena.allocBytes(T * latent_q * es);
    b.latent_rows = arena.allocBytes(rows * expand_rank * es);
    b.latent_products = arena.allocBytes(rows * expand_n * es);
    b.latent_pages = arena.allocBytes(b.latent_max_pages * expand_page * es);
    b.latent_page_ids = (int32_t*)arena.allocBytes((size_t)m.kv_pages * 4);
  }
  for (int32_t** p : {&b.routing.choice, &b.routing.place, &b.routing.row_of}) *p = (int32_t*)arena.allocBytes(T * top * 4);
  for (float** p : {&b.routing.weight, &b.routing.row_weight}) *p = (float*)arena.allocBytes(T * top * 4);
  b.routing.offsets = (int32_t*)arena.allocBytes((experts + 1) * 4);
  b.routing.tile_group = (int32_t*)arena.allocBytes(tiles * 4);
  b.routing.tile_row = (int32_t*)arena.allocBytes(tiles * 4);
  b.routing.n_tiles = (int32_t*)arena.allocBytes(4);
  b.router_sums = (float*)arena.allocBytes(b.router_sums_bytes);
  b.expert_ff = arena.allocBytes(T * expert_ff * es);
  b.expert_out = arena.allocBytes(T * top * ld * es);
  b.side_sums = (float*)arena.allocBytes(b.side_sums_bytes);
  b.side = arena.allocBytes(T * side * es);
  b.y = bf16 && T > kSumsMaxRows ? arena.allocBytes(T * ld * es) : nullptr;
  b.y_sums = (float*)arena.allocBytes(b.y_sums_bytes);
  b.ff = arena.allocBytes(T * ff * es);
  b.head_in = arena.allocBytes(L * ld * es);
  b.logits = (float*)arena.allocBytes(b.logits_bytes);
  b.argmax = (int32_t*)arena.allocBytes((size_t)L * 4);
  b.gemm_ws = arena.allocBytes(b.gemm_ws_bytes);
  b.gemm_ws_side = arena.allocBytes(b.gemm_ws_bytes);
  b.recur_ws = arena.allocBytes(recur);
  b.latent_ws = arena.allocBytes(b.latent_ws_bytes);
  return b;
}

size_t LayerStackPipeline::tmpBytes(const StackModel& m, int max_rows) {
  AllocationManager<half> count((half*)nullptr, (size_t)1 << 46);  // addresses only
  (void)plan(m, max_rows, count);
  return count.getAllocation() * sizeof(half);
}

void LayerStackPipeline::config(vortexConfigData* config_data_) {
  clearGraphs();
  config_error.clear();
  this->config_data = *config_data_;
  const int T = config_data.global_batch_size;
  if (T <= 0 || T > ModelConfig.max_batch_size) {
    configFail("LayerStackPipeline::config: global batch %d not in (0, %d]", T, ModelConfig.max_batch_size);
    return;
  }
  AllocationManager<half> arena(input_data->tmp_buffer, input_data->tmp_buffer_size);
  buf = plan(*model, T, arena);
  // columns past a row's true width are never written and must read as zero
  HIP_CHECK(hipMemset(input_data->tmp_buffer, 0, arena.getAllocation() * sizeof(half)));
  if (layer_outputs) (void)hipFree(layer_outputs);
  layer_outputs = nullptr;
  const StackModelSpec& spec = model->spec;
  const int ld = spec.ld();
  if (keep_layers) HIP_CHECK(hipMalloc(&layer_outputs, model->runs.size() * (size_t)T * ld * sizeof(float)));

  for (StackOperator* op : std::initializer_list<StackOperator*>{&embedding, &linear, &firstNorm, &residualAdd, &grouped, &router,
                                                                 &tokenGate, &gatedNorm, &latentAppend, &latentAttention, &latentExpand, &latentQueries, &tokenShift,
                                                                 &tanhRows, &qkvAppend, &attention, &recurrence, &gatherNorm, &sampler}) {
    op->setStream(stream_all);
    op->batch = &batch;
    op->dtype = model->dtype;
  }
  linear_side.setStream(stream_side);
  linear_side.batch = &batch;
  linear_side.dtype = model->dtype;
  linear.workspace = buf.gemm_ws;
  linear_side.workspace = buf.gemm_ws_side;
  linear.workspace_bytes = linear_side.workspace_bytes = buf.gemm_ws_bytes;
  embedding.w = &model->weights;
  embedding.x = buf.x;
  // where a norm comes first the rows themselves are not read, and in fp32 they are x
  embedding.act = model->dtype == NF_BF16 && !spec.pre_norm ? buf.act : nullptr;
  embedding.ld = ld;
  embedding.scale = (float)spec.embedding_scale;
  firstNorm.x = buf.x;
  firstNorm.norm = model->weights.layers[0].norm1;
  firstNorm.out = buf.act;
  residualAdd.args.x = buf.x;
  residualAdd.args.y_scale = (float)spec.residual_scale;
  residualAdd.args.width = gatherNorm.width = firstNorm.width = spec.width;
  residualAdd.args.ld = gatherNorm.ld = tokenShift.ld = firstNorm.ld = ld;
  qkvAppend.eps = latentAppend.eps = gatedNorm.eps = (float)spec.eps;
  tokenShift.x = buf.x;
  tokenShift.out = buf.mix;
  gatherNorm.x = buf.x;
  gatherNorm.norm = model->weights.final_norm;
  gatherNorm.out = buf.head_in;
  sampler.logits = buf.logits;
  sampler.argmax = buf.argmax;
  sampler.cols = spec.vocab;
  sampler.ld = model->weights.head.N;
  setName();

  delete[] output_data.sampled_token_array;
  output_data = vortexOutputData();
  output_data.sampled_token_array = new int[T]();
  output_data.global_batch_size = T;
  if (profiling) setProfiling(profilingLevel());
}

void LayerStackPipeline::setName() {
  SET_NAME_REF(embedding);
  SET_NAME_REF(linear);
  SET_NAME_REF(linear_side);
  SET_NAME_REF(firstNorm);
  SET_NAME_REF(residualAdd);
  SET_NAME_REF(grouped);
  SET_NAME_REF(router);
  SET_NAME_REF(tokenGate);
  SET_NAME_REF(gatedNorm);
  SET_NAME_REF(latentAppend);
  SET_NAME_REF(latentAttention);
  SET_NAME_REF(latentExpand);
  SET_NAME_REF(latentQueries);
  SET_NAME_REF(tokenShift);
  SET_NAME_REF(tanhRows);
  SET_NAME_REF(qkvAppend);
  SET_NAME_REF(attention);
  SET_NAME_REF(recurrence);
  SET_NAME_REF(gatherNorm);
  SET_NAME_REF(sampler);
}

void LayerStackPipeline::setProfiling(int level) {
  profiling = level > 0;
  profile_gemms = level > 1;
  const unsigned stride = profileStride();
  timings.layer_stride = (int)stride;
  const size_t n = model->runs.size();
  attention.enableProfiling(profiling ? n : 0, stride);
  latentAttention.enableProfiling(profiling ? n : 0, stride);
  linear.enableProfiling(profile_gemms ? 10 * n + 1 : 0, 1);
  linear_side.enableProfiling(profile_gemms ? n : 0, 1);
}

void LayerStackPipeline::update(vortexUpdateData* u) {
  this->update_data = *u;
  batch.decode = u->decodePrefillBorder;
  batch.prefill = u->prefillNum;
  batch.rows = u->decodePrefillBorder + u->prefillTokensNum;
  batch.logit_rows = u->logit_rows_num;
  batch.tokens = u->input_tokens;
  batch.positions = u->per_token_offset;
  batch.input_indptr = u->input_indptr;
  batch.rev_input_indptr = u->rev_input_indptr;
  batch.kv_indptr = u->kv_indptr;
  batch.kv_indices = u->kv_indices;
  batch.state_slots = u->state_slots;
  batch.logit_row_index = u->logit_rows;
  output_data.sampled_tokens = batch.logit_rows;
}

// What the first sublayer of a run reads, and what comes ahead of it.
LayerStackPipeline::Next LayerStackPipeline::beforeRun(int run) const {
  const LayerRun& r = model->runs[run];
  Next n{true, {}, r.enters};
  if (model->spec.pre_norm) n.norm = model->weights.layers[r.layer].norm1;
  return n;
}

LayerStackPipeline::Next LayerStackPipeline::afterLayer(int run) const {
  if (run + 1 == (int)model->runs.size()) return {};  // the last norm takes the rows that are wanted
  // the stream as a layer leaves it is copied out before anything else is added
  if (layer_outputs && model->runs[run + 1].enters >= 0) return {};
  return beforeRun(run + 1);
}

LayerStackPipeline::Next LayerStackPipeline::afterFeedForward(int run) const {
  return model->spec.token_side > 0 ? Next{true, {}} : afterLayer(run);
}

LayerStackPipeline::Next LayerStackPipeline::afterMixer(int run) const {
  const int layer = model->runs[run].layer;
  if (!model->spec.layers[layer].hasFeedForward()) return afterFeedForward(run);
  return model->spec.pre_norm ? Next{true, model->weights.layers[layer].norm2} : Next{true, {}};
}

void LayerStackPipeline::setNext(const Next& next) {
  nf_residual_args& r = residualAdd.args;
  r.add = next.enters >= 0 ? model->weights.loop_step + (size_t)next.enters * model->spec.ld() : nullptr;
  r.table = next.enters > 0 ? model->weights.embed.ptr : nullptr;
  r.table_scale = (float)model->spec.embedding_scale;
  residualAdd.args.next = next.norm;
  // in fp32 the residual stream is its own plain form
  const bool written = next.wanted && (next.norm.kind != NF_NORM_NONE || model->dtype == NF_BF16);
  residualAdd.args.act = written ? buf.act : nullptr;
}

// What comes ahead of a run that no sublayer's end has left.
void LayerStackPipeline::enterRun(int run) {
  nf_residual_args& r = residualAdd.args;
  r.y = nullptr;
  r.routing = nullptr;
  r.y_norm = nf_norm{};
  setNext(beforeRun(run));
  residualAdd.run();
}

// Projection back to the residual width, norm, residual add, what the next sublayer reads.
void LayerStackPipeline::sublayerOut(const void* a, const DeviceMatrix& w, const nf_norm& y_norm, const Next& next) {
  nf_residual_args& r = residualAdd.args;
  r.routing = nullptr;
  r.y_norm = y_norm;
  if (model->dtype == NF_BF16 && batch.rows > kSumsMaxRows &&
      nf_gemm_nk_sums_shares(batch.rows, w.N, w.K, kSumsMaxShares) < 2) {
    linear.set(a, w, buf.y, batch.rows).run();
    r.y = buf.y;
    r.y_dtype = NF_BF16;
    r.shares = 1;
  } else {
    linear.setSums(a, w, buf.y_sums, buf.y_sums_bytes, batch.rows, kSumsMaxShares).run();
    r.y = buf.y_sums;
    r.y_dtype = NF_F32;
    r.shares = linear.shares();
  }
  setNext(next);
  residualAdd.run();
}

// Router, the chosen experts' feed-forwards, their weighted sum added to the residual stream.
void LayerStackPipeline::mixtureOut(int run) {
  const int layer = model->runs[run].layer;
  const MixtureSpec& s = *model->spec.layers[layer].mixture;
  const LayerWeights& w = model->weights.layers[layer];
  const int T = batch.rows, experts = s.experts + s.always(), slots = T * s.perToken(), ld = model->spec.ld();
  const void* h = sublayerInput();
  linear.setSums(h, w.router, buf.router_sums, buf.router_sums_bytes, T, kSumsMaxShares).run();
  nf_route_args& z = router.args;
  z.z = buf.router_sums;
  z.shares = linear.shares();
  z.ld = w.router.N;
  z.outputs = s.outputs();
  z.experts = s.experts;
  z.top = s.top;
  z.always = s.always();
  z.groups = s.groups;
  z.keep_groups = s.keep_groups;
  z.correction = w.correction;
  z.scale = (float)s.scale;
  z.scores = s.scores;
  z.always_plain = !s.shared_gate;
  router.routing = buf.routing;
  if (!s.weigh_input) router.routing.row_weight = nullptr;
  router.routing.tile_rows = nf_grouped_tile_rows(model->dtype, slots, experts);
  router.run();
  const int ff = w.down.K;
  grouped.experts(h, ld, w.up, buf.expert_ff, ff, experts, router.routing, true, slots, s.gated ? NF_ACT_GATED : s.act);
  grouped.args.weigh = s.weigh_input;
  if (s.gated) grouped.args.gated = nf_gated_act{(float)s.gated->slope, (float)s.gated->shift, w.limits};
  grouped.run();
  grouped.experts(buf.expert_ff, ff, w.down, buf.expert_out, ld, experts, router.routing, false, slots, NF_ACT_NONE);
  grouped.run();
  nf_residual_args& r = residualAdd.args;
  nf_routing places = router.routing;
  if (s.weigh_input) places.weight = nullptr;  // it has been in the experts' inputs
  r.routing = &places;
  r.y = buf.expert_out;
  r.y_ld = ld;
  r.top = s.perToken();
  r.identity = s.identity > 0 ? h : nullptr;
  r.y_norm = w.out_norm2;
  setNext(afterFeedForward(run));
  residualAdd.run();
  r.routing = nullptr;
}

// The layer's input for the tokens themselves.
void LayerStackPipeline::tokenSide(int run) {
  const int layer = model->runs[run].layer;
  const LayerWeights& w = model->weights.layers[layer];
  linear.setSums(plain(), w.side_gate, buf.side_sums, buf.side_sums_bytes, batch.rows, kSumsMaxShares).run();
  tokenGate.sums = buf.side_sums;
  tokenGate.shares = linear.shares();
  tokenGate.table = model->weights.side_embed.ptr;
  tokenGate.table_ld = model->weights.side_embed.K;
  tokenGate.dim = model->spec.token_side;
  tokenGate.col0 = layer * tokenGate.dim;
  tokenGate.out = buf.side;
  tokenGate.cols = w.side_gate.N;
  tokenGate.run();
  sublayerOut(buf.side, w.side_proj, w.side_norm, afterLayer(run));
}

// Pages of keys and values to write out for the prompts of a layer with latent attention; 0: attend over the latents.  Counted in
// multiplications per head: writing out costs its product per token of context and saves, per row, the two products with the
// row and the difference of the two forms' widths per key it sees.
int LayerStackPipeline::expandPages(int layer) const {
  if (batch.prefill == 0 || model->expandedLayout(layer).page == 0) return 0;
  const LatentAttentionSpec& s = *model->spec.layers[layer].latent;
  const LatentAttentionWeights& w = model->weights.layers[layer].latent;
  const nf_latent_layout l = model->latentLayout(layer);
  const int32_t *kv = host_update_data.kv_indptr, *in = host_update_data.input_indptr;
  const int first = batch.decode, end = batch.decode + batch.prefill;
  const int pages = (kv[end] - kv[first] + kExpandGroup - 1) / kExpandGroup * kExpandGroup;
  if (pages > buf.latent_max_pages) return 0;
  double pairs = 0;
  for (int r = first; r < end; ++r) {
    const double rows = in[r + 1] - in[r], context = (double)(kv[r + 1] - kv[r]) * model->page_size;
    const double seen = std::max(context - rows / 2, rows / 2);
    pairs += rows * (s.window > 0 ? std::min(seen, (double)s.window) : seen);
  }
  const double product = (double)l.rank_pad * (w.dim_pad + w.vdim_pad), tokens = (double)(kv[end] - kv[first]) * model->page_size;
  const double saved = pairs * (l.row_ld + l.rank_pad - (w.dim_pad + s.rot_dim + w.vdim_pad)) + (batch.rows - batch.decode) * product;
  return saved > tokens * product ? pages : 0;
}

void LayerStackPipeline::latentBranch(int run) {
  const int layer = model->runs[run].layer;
  const LatentAttentionSpec& s = *model->spec.layers[layer].latent;
  const LayerWeights& lw = model->weights.layers[layer];
  const LatentAttentionWeights& w = lw.latent;
  const nf_latent_layout l = model->latentLayout(layer);
  linear.set(sublayerInput(), w.proj, buf.attn_proj, batch.rows).run();
  latentAppend.layout = l;
  latentAppend.proj = buf.attn_proj;
  latentAppend.w = &w;
  latentAppend.q = buf.q;
  latentAppend.kv_data = model->kv_data[run];
  // rows that attend over the latents: all of them, or the decode rows
  const int pages = expandPages(layer), rows = pages > 0 ? batch.decode : batch.rows;
  latentAppend.q_rows = rows;
  latentAppend.run();
  if (pages > 0) {
    nf_latent_expand_args& x = latentExpand.args;
    x.layout = l;
    x.kv = model->expandedLayout(layer);
    x.dim_pad = w.dim_pad;
    x.kv_data = model->kv_data[run];
    x.kv_indptr = batch.kv_indptr;
    x.kv_indices = batch.kv_indices;
    x.req_begin = batch.decode;
    x.req_end = batch.decode + batch.prefill;
    x.max_pages = pages;
    x.rows = buf.latent_rows;
    x.page_ids = buf.latent_page_ids;
    x.products = buf.latent_products;
    x.ld = w.expand.N;
    x.k_col = 0;
    x.v_col = s.heads * w.dim_pad;
    x.pages = buf.latent_pages;
    latentExpand.product = &linear;
    latentExpand.w = &w;
    latentExpand.run();
    latentQueries.kv = x.kv;
    latentQueries.proj = buf.attn_proj;
    latentQueries.w = &w;
    latentQueries.rot_dim = s.rot_dim;
    latentQueries.q = buf.latent_q;
    latentQueries.run();
    nf_window_attention_args& g = attention.args;
    g = nf_window_attention_args{};
    g.kv = x.kv;
    g.window = s.window;
    g.scale = (float)s.scale;
    g.out_scale = 1.f;
    g.q = buf.latent_q;
    g.out = buf.heads;
    g.out_ld = lw.out.K;
    g.kv_data = buf.latent_pages;
    attention.setStream(stream_all);
    attention.page_ids = buf.latent_page_ids;
    attention.decoding = false;
    attention.run();
    attention.page_ids = nullptr;
    attention.decoding = true;
  }
  if (rows == 0) return;
  grouped.heads(rows, buf.attn_proj, w.proj.N, w.dim_pad, w.to_latent, buf.q, s.heads * l.row_ld, l.row_ld, s.heads);
  grouped.run();
  nf_latent_attention_args& a = latentAttention.args;
  a.layout = l;
  a.window = s.window;
  a.scale = (float)s.scale;
  a.q = buf.q;
  a.out = buf.latent;
  a.kv_data = model->kv_data[run];
  a.workspace = buf.latent_ws;
  a.workspace_bytes = buf.latent_ws_bytes;
  latentAttention.prompts = pages == 0;
  latentAttention.run();
  grouped.heads(rows, buf.latent, s.heads * l.rank_pad, l.rank_pad, w.from_latent, buf.heads, lw.out.K, w.vdim_pad, s.heads);
  grouped.run();
}

void LayerStackPipeline::attentionBranch(int run, hipStream_t s) {
  const int layer = model->runs[run].layer;
  const AttentionSpec& a = *model->spec.layers[layer].attention;
  const LayerWeights& w = model->weights.layers[layer];
  linear_side.setStream(s);
  qkvAppend.setStream(s);
  attention.setStream(s);
  linear_side.set(sublayerInput(), w.attention.qkv, buf.attn_proj, batch.rows, NF_ACT_NONE, w.attention.bias).run();
  qkvAppend.kv = model->kvLayout(layer);
  qkvAppend.proj = buf.attn_proj;
  qkvAppend.ld = w.attention.qkv.N;
  qkvAppend.w = &w.attention;
  qkvAppend.q_temp.reset();
  if (a.q_temp) qkvAppend.q_temp = nf_query_temperature{(float)a.q_temp->coef, a.q_temp->every};
  qkvAppend.value_norm = a.value_norm;
  qkvAppend.conv_taps = a.conv_taps;
  qkvAppend.conv_state = model->conv_state[run];
  qkvAppend.q_out = buf.q;
  qkvAppend.kv_data = model->kv_data[run];
  qkvAppend.run();
  nf_window_attention_args& g = attention.args;
  g.kv = qkvAppend.kv;
  g.window = a.window;
  g.keep_first = a.keep_first;
  g.chunk = a.chunk;
  g.out_rot = w.attention.value_rot;
  g.scale = (float)a.scale;
  g.out_scale = (float)a.out_scale;
  g.softcap = (float)a.softcap;
  g.map_weight = w.attention.map_weight;
  g.head_norm = a.head_norm;
  g.head_eps = (float)model->spec.eps;
  g.sink = w.attention.sink;
  g.gate = a.head_gate ? (const uint8_t*)buf.attn_proj + (size_t)w.attention.g_col * model->elementBytes() : nullptr;
  g.gate_ld = qkvAppend.ld;
  g.q = buf.q;
  g.out = buf.heads;
  g.out_ld = w.out.K;
  g.out_col = 0;
  g.kv_data = model->kv_data[run];
  attention.run();
}

void LayerStackPipeline::recurrenceBranch(int run) {
  const int layer = model->runs[run].layer;
  const LayerSpec& spec = model->spec.layers[layer];
  const RecurrenceSpec& r = *spec.recurrence;
  const LayerWeights& lw = model->weights.layers[layer];
  const RecurrenceWeights& w = lw.recurrence;
  const int T = batch.rows;
  const size_t es = model->elementBytes();
  auto at = [&](const void* p, int col) { return (const void*)((const uint8_t*)p + (size_t)col * es); };
  nf_recurrence_args& a = recurrence.args;
  a = nf_recurrence_args{};
  a.dtype = model->dtype;
  a.kind = r.kind;
  a.heads = r.heads;
  a.dim = r.dim;
  a.vdim = r.vdim;
  if (r.kind == NF_RECURRENCE_FIXED_DECAY) {
    linear.set(sublayerInput(), w.qkvg, buf.mix, T, r.qkv_act).run();
    a.q = at(buf.mix, w.q_col);
    a.k = at(buf.mix, w.k_col);
    a.v = at(buf.mix, w.v_col);
    a.g = at(buf.mix, w.g_col);
    a.q_ld = a.k_ld = a.v_ld = a.g_ld = w.qkvg.N;
    if (w.g.N > 0) {
      linear.set(sublayerInput(), w.g, buf.rkvg[3], T).run();
      a.g = buf.rkvg[3];
      a.g_ld = w.g.N;
    }
    a.rot = w.rot;
    a.k_scale = (float)r.k_scale;
    a.log2_decay = w.log2_decay;
  } else {
    tokenShift.shift_state = model->shift_state[run];
    tokenShift.mu = w.mu;
    tokenShift.run();
    auto mixed = [&](int s) { return (const void*)((const uint8_t*)buf.mix + (size_t)s * T * tokenShift.ld * es); };
    const DeviceMatrix* in[4] = {&w.r, &w.k, &w.v, &w.g};
    for (int i = 0; i < 4; ++i) linear.set(mixed(i), *in[i], buf.rkvg[i], T).run();
    linear.setSums(mixed(4), w.w1, buf.w1_sums, buf.w1_sums_bytes, T, kSumsMaxShares).run();
    tanhRows.sums = buf.w1_sums;
    tanhRows.shares = linear.shares();
    tanhRows.cols = w.w1.N;
    tanhRows.out = buf.w1_act;
    tanhRows.run();
    linear.setSums(buf.w1_act, w.w2, buf.z, buf.z_bytes, T, 1).run();
    a.q = buf.rkvg[0];
    a.k = buf.rkvg[1];
    a.v = buf.rkvg[2];
    a.g = buf.rkvg[3];
    a.q_ld = w.r.N;
    a.k_ld = w.k.N;
    a.v_ld = w.v.N;
    a.g_ld = w.g.N;
    a.z = buf.z;
    a.z_ld = w.w2.N;
    a.z_shares = 1;
    a.w0 = w.w0;
    a.u = w.u;
    a.norm_weight = w.norm;
    a.shift_x = buf.x;
    a.shift_state = model->shift_state[run];
    a.shift_ld = tokenShift.ld;
  }
  a.eps = (float)model->spec.eps;
  a.out_scale = (float)r.out_scale;
  a.state = model->state[run];
  a.out = buf.heads;
  a.out_ld = lw.out.K;
  a.out_col = spec.attention ? spec.attention->heads * spec.attention->vdim : 0;
  a.workspace = buf.recur_ws;
  a.workspace_bytes = buf.recur_ws_bytes;
  if (r.joint_norm) {  // the heads as the recurrence leaves them
    gatedNorm.g = a.g;
    gatedNorm.g_ld = a.g_ld;
    a.g = nullptr;
  }
  recurrence.run();
  if (r.joint_norm) {
    gatedNorm.o = (uint8_t*)buf.heads + (size_t)a.out_col * es;
    gatedNorm.o_ld = a.out_ld;
    gatedNorm.weight = w.norm;
    gatedNorm.width = r.heads * r.vdim;
    gatedNorm.run();
  }
}

void LayerStackPipeline::enqueueMixer(int run) {
  const int layer = model->runs[run].layer;
  const LayerSpec& s = model->spec.layers[layer];
  const bool both = s.attention && s.recurrence;
  if (both) {  // two mixers that read the same rows and write different columns
    HIP_CHECK(hipEventRecord(fork, stream_all));
    HIP_CHECK(hipStreamWaitEvent(stream_side, fork, 0));
    attentionBranch(run, stream_side);
    HIP_CHECK(hipEventRecord(join, stream_side));
  } else if (s.attention) {
    attentionBranch(run, stream_all);
  }
  if (s.latent) latentBranch(run);
  if (s.recurrence) recurrenceBranch(run);
  if (both) HIP_CHECK(hipStreamWaitEvent(stream_all, join, 0));
  const LayerWeights& w = model->weights.layers[layer];
  sublayerOut(buf.heads, w.out, w.out_norm1, afterMixer(run));
}

void LayerStackPipeline::enqueueIteration() {
  const StackModelSpec& spec = model->spec;
  embedding.run();
  if (spec.pre_norm && model->runs[0].enters < 0) firstNorm.run();
  for (int run = 0; run < (int)model->runs.size(); ++run) {
    const LayerSpec& layer = spec.layers[model->runs[run].layer];
    const LayerWeights& w = model->weights.layers[model->runs[run].layer];
    if (model->runs[run].enters >= 0 && (run == 0 || layer_outputs)) enterRun(run);
    enqueueMixer(run);
    if (layer.mlp) {
      linear.set(sublayerInput(), w.up, buf.ff, batch.rows, layer.mlp->act).run();
      sublayerOut(buf.ff, w.down, w.out_norm2, afterFeedForward(run));
    }
    if (layer.mixture) mixtureOut(run);
    if (spec.token_side > 0) tokenSide(run);
    if (layer_outputs)
      HIP_CHECK(hipMemcpyAsync(layer_outputs + (size_t)run * config_data.global_batch_size * spec.ld(), buf.x,
                               (size_t)batch.rows * spec.ld() * sizeof(float), hipMemcpyDeviceToDevice, stream_all));
  }
  if (batch.logit_rows == 0) return;
  gatherNorm.run();
  linear.setSums(buf.head_in, model->weights.head, buf.logits, buf.logits_bytes, batch.logit_rows, 1).run();
  sampler.run();
}

vortexOutputData LayerStackPipeline::run() {
  HIP_CHECK(hipEventRecord(events[EventManager::GEMM_TIMING_START], stream_all));
  std::vector<int> sig = baseSignature();
  sig.push_back(batch.logit_rows);
  for (const LayerRun& r : model->runs)
    if (model->spec.layers[r.layer].latent) sig.push_back(expandPages(r.layer));
  if (layer_outputs) {
    ++graph_eager;
    enqueueIteration();
  } else {
    runIteration(stream_all, sig, [this] { enqueueIteration(); });
  }
  HIP_CHECK(hipEventRecord(events[EventManager::GEMM_TIMING_END], stream_all));
  if (batch.logit_rows > 0)
    HIP_CHECK(hipMemcpyAsync(output_data.sampled_token_array, buf.argmax, batch.logit_rows * sizeof(int), hipMemcpyDeviceToHost,
                             stream_all));
  HIP_CHECK(hipStreamSynchronize(stream_all));
  float ms = 0;
  HIP_CHECK(hipEventElapsedTime(&ms, events[EventManager::GEMM_TIMING_START], events[EventManager::GEMM_TIMING_END]));
  timings.iter_ms = ms;
  if (profiling) {
    // one attention operator launches for the decode rows and for the prompts
    double& t = batch.decode > 0 ? timings.decode_attn_ms : timings.prefill_attn_ms;
    long& n = batch.decode > 0 ? timings.decode_attn_launches : timings.prefill_attn_launches;
    attention.collectProfile(t, n);
    latentAttention.collectProfile(t, n);
  }
  if (profile_gemms) {
    linear.collectProfile(timings.gemm_ms, timings.gemm_launches);
    linear_side.collectProfile(timings.gemm_ms, timings.gemm_launches);
  }
  return output_data;
}
