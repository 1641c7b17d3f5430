// Operators of the layer-stack pipeline over the kernel layer's C ABI (nf_route ... nf_linear_recurrence),
// in the vocabulary of OperatorWrapper: a stream, run(), per-launch timing.
#pragma once
#include "operatorWrapper.h"
#include "stackModel.h"

// The iteration's device arrays (TensorManager's mirrors) and the integers that shape its launches.
struct StackBatch {
  int rows = 0;         // tokens
  int decode = 0;       // requests [0, decode) have one row each, rows [0, decode)
  int prefill = 0;      // requests [decode, decode + prefill): portions of prompts
  int logit_rows = 0;   // rows the head computes
  const int32_t *tokens = nullptr, *positions = nullptr, *input_indptr = nullptr, *rev_input_indptr = nullptr;
  const int32_t *kv_indptr = nullptr, *kv_indices = nullptr, *state_slots = nullptr, *logit_row_index = nullptr;
};

struct StackOperator : public OperatorWrapper {
  const StackBatch* batch = nullptr;
  nf_dtype dtype = NF_BF16;
  StackOperator() : OperatorWrapper(false, false) {}
};

// D = act(A . W^T + bias).  The output is rounded to the activations' type, or left as fp32 sums in shares of K
// for an operator that adds them (sums()).
struct StackLinear : public StackOperator {
  const void* a = nullptr;
  void* d = nullptr;
  DeviceMatrix w;
  const void* bias = nullptr;
  nf_activation act = NF_ACT_NONE;
  int rows = 0;
  bool as_sums = false;
  int max_shares = 1;
  size_t d_bytes = 0;  // of a sums buffer
  void* workspace = nullptr;
  size_t workspace_bytes = 0;

  StackLinear& set(const void* a_, const DeviceMatrix& w_, void* d_, int rows_, nf_activation act_ = NF_ACT_NONE,
                   const void* bias_ = nullptr) {
    bias = bias_;
    a = a_;
    w = w_;
    d = d_;
    rows = rows_;
    act = act_;
    as_sums = false;
    return *this;
  }
  StackLinear& setSums(const void* a_, const DeviceMatrix& w_, void* d_, size_t bytes, int rows_, int max_shares_) {
    set(a_, w_, d_, rows_);
    as_sums = true;
    d_bytes = bytes;
    max_shares = max_shares_;
    return *this;
  }
  int shares() const {
    return as_sums && dtype == NF_BF16 ? nf_gemm_nk_sums_shares(rows, w.N, w.K, max_shares) : 1;
  }
  double totalCompute() const { return 2.0 * rows * (double)w.N * w.K; }
  void work() override {
    if (dtype == NF_F32) {
      NF_KERNEL_CHECK(nf_gemm_nk_f32((const float*)a, (const float*)w.ptr, (const float*)bias, (float*)d, rows, w.N, w.K, act, stream));
    } else if (as_sums) {
      NF_KERNEL_CHECK(nf_gemm_nk_sums_bf16((const uint16_t*)a, (const uint16_t*)w.ptr, (float*)d, d_bytes, rows, w.N, w.K,
                                           max_shares, stream));
    } else if (bias) {
      NF_KERNEL_CHECK(nf_gemm_nk_bias_bf16((const uint16_t*)a, (const uint16_t*)w.ptr, (const uint16_t*)bias, (uint16_t*)d, rows, w.N, w.K,
                                           workspace, workspace_bytes, stream));
    } else {
      auto f = act == NF_ACT_SQUARED_RELU ? nf_gemm_nk_relu2_bf16 : act == NF_ACT_SILU ? nf_gemm_nk_silu_bf16 : act == NF_ACT_GELU ? nf_gemm_nk_gelu_bf16 : nf_gemm_nk_bf16;
      NF_KERNEL_CHECK(f((const uint16_t*)a, (const uint16_t*)w.ptr, (uint16_t*)d, rows, w.N, w.K, workspace, workspace_bytes,
                        stream));
    }
  }
};

struct StackEmbedding : public StackOperator {
  const StackWeights* w = nullptr;
  float* x = nullptr;
  void* act = nullptr;
  int ld = 0;
  float scale = 1;
  void work() override {
    NF_KERNEL_CHECK(nf_embed_rows(dtype, batch->tokens, batch->positions, w->embed.ptr, w->pos.ptr, scale, x, act, batch->rows, ld, stream));
  }
};

// The norm ahead of the first sublayer.
struct StackNorm : public StackOperator {
  const float* x = nullptr;
  nf_norm norm{};
  void* out = nullptr;
  int width = 0, ld = 0;
  void work() override { NF_KERNEL_CHECK(nf_norm_rows(dtype, x, nullptr, &norm, out, batch->rows, width, ld, stream)); }
};

// The end of a sublayer: its output, normed or put together from experts, added to the residual stream, what a pass over
// layers starts with, and what the next sublayer reads.
struct StackResidual : public StackOperator {
  nf_residual_args args{};
  void work() override {
    nf_residual_args a = args;
    a.rows = batch->rows;
    a.dtype = dtype;
    a.tokens = batch->tokens;
    NF_KERNEL_CHECK(nf_residual_rows(&a, stream));
  }
};

// Products with a group of weights each: heads (every group has all rows), or experts (the routing's rows).
struct StackGroupedLinear : public StackOperator {
  nf_grouped_gemm_args args{};
  int rows = 0;
  void heads(int rows_, const void* a, int lda, size_t a_group, const DeviceMatrix& w, void* d, int ldd, size_t d_group, int groups) {
    rows = rows_;
    args = nf_grouped_gemm_args{};
    args.groups = groups;
    args.a = a;
    args.lda = lda;
    args.a_group = a_group;
    args.d_group = d_group;
    set(w, d, ldd);
  }
  void experts(const void* a, int lda, const DeviceMatrix& w, void* d, int ldd, int groups, const nf_routing& r, bool gather, int max_rows,
               nf_activation act) {
    rows = batch->rows;
    args = nf_grouped_gemm_args{};
    args.groups = groups;
    args.a = a;
    args.lda = lda;
    args.routing = r;
    args.gather = gather;
    args.max_rows = max_rows;
    args.act = act;
    set(w, d, ldd);
  }
  void work() override {
    args.dtype = dtype;
    args.M = rows;
    NF_KERNEL_CHECK(nf_gemm_grouped(&args, stream));
  }

private:
  void set(const DeviceMatrix& w, void* d, int ldd) {
    args.b = w.ptr;
    args.N = w.N;
    args.K = w.K;
    args.d = d;
    args.ldd = ldd;
  }
};

struct StackRouter : public StackOperator {
  nf_route_args args{};
  nf_routing routing{};
  void work() override {
    args.rows = batch->rows;
    NF_KERNEL_CHECK(nf_route(&args, &routing, stream));
  }
};

struct StackTokenGate : public StackOperator {
  const float* sums = nullptr;
  int shares = 1, table_ld = 0, col0 = 0, dim = 0, cols = 0;
  const void* table = nullptr;
  void* out = nullptr;
  void work() override {
    NF_KERNEL_CHECK(nf_token_gate_rows(dtype, sums, shares, batch->tokens, table, table_ld, col0, dim, out, batch->rows, cols, stream));
  }
};

struct StackGatedNorm : public StackOperator {
  void* o = nullptr;
  const void* g = nullptr;
  int o_ld = 0, g_ld = 0, width = 0;
  const float* weight = nullptr;
  float eps = 0;
  void work() override { NF_KERNEL_CHECK(nf_gated_norm_rows(dtype, o, o_ld, g, g_ld, weight, batch->rows, width, eps, stream)); }
};

struct StackTokenShift : public StackOperator {
  const float *x = nullptr, *shift_state = nullptr, *mu = nullptr;
  void* out = nullptr;
  int n_mix = 5, ld = 0;
  void work() override {
    NF_KERNEL_CHECK(nf_token_shift(dtype, x, shift_state, mu, out, n_mix, batch->input_indptr, batch->rev_input_indptr,
                                   batch->positions, batch->state_slots, batch->rows, ld, stream));
  }
};

struct StackTanh : public StackOperator {
  const float* sums = nullptr;
  int shares = 1, cols = 0;
  void* out = nullptr;
  void work() override { NF_KERNEL_CHECK(nf_tanh_rows(dtype, sums, shares, out, batch->rows, cols, stream)); }
};

struct StackLatentAppend : public StackOperator {
  nf_latent_layout layout{};
  const void* proj = nullptr;
  const LatentAttentionWeights* w = nullptr;
  float eps = 0;
  int q_rows = 0;
  void *q = nullptr, *kv_data = nullptr;
  void work() override {
    NF_KERNEL_CHECK(nf_latent_append(&layout, proj, w->proj.N, w->q_col, w->kv_col, w->norm, eps, &w->rot, q, kv_data, batch->kv_indptr,
                                     batch->kv_indices, batch->rev_input_indptr, batch->positions, batch->rows, q_rows, stream));
  }
};

// The latents behind the prompts' portions as keys and values of all heads, in pages of their own.
struct StackLatentExpand : public StackOperator {
  nf_latent_expand_args args{};
  StackLinear* product = nullptr;
  const LatentAttentionWeights* w = nullptr;
  void work() override {
    NF_KERNEL_CHECK(nf_latent_gather(&args, stream));
    product->set(args.rows, w->expand, const_cast<void*>(args.products), args.max_pages * 16).run();
    NF_KERNEL_CHECK(nf_latent_pack(&args, stream));
  }
};
struct StackLatentQueries : public StackOperator {
  nf_kv_layout kv{};
  const void* proj = nullptr;
  const LatentAttentionWeights* w = nullptr;
  int rot_dim = 0;
  void* q = nullptr;
  void work() override {
    NF_KERNEL_CHECK(nf_latent_queries(&kv, w->dim_pad, proj, w->proj.N, w->q_col, rot_dim, &w->rot, batch->positions, q, batch->decode,
                                      batch->rows - batch->decode, stream));
  }
};

// Short convolution, per-head norm and rotation of projected rows, append to the paged cache (the counterpart of
// RoPEAppend); the convolution's state.
struct StackQKVAppend : public StackOperator {
  nf_kv_layout kv{};
  const void* proj = nullptr;
  int ld = 0;
  const AttentionWeights* w = nullptr;
  float eps = 0;
  std::optional<nf_query_temperature> q_temp;
  bool value_norm = false;
  int conv_taps = 0;
  void* conv_state = nullptr;
  void *q_out = nullptr, *kv_data = nullptr;
  void work() override {
    const nf_value_form values{value_norm, w->value_rot};
    const nf_short_conv conv{conv_taps, w->conv, conv_state, batch->input_indptr, batch->state_slots};
    NF_KERNEL_CHECK(nf_qkv_append(&kv, proj, ld, w->q_col, w->k_col, w->v_col, w->q_norm, w->k_norm, eps, &w->rot,
                                  q_temp ? &*q_temp : nullptr, &values, conv_taps > 0 ? &conv : nullptr, q_out, kv_data, batch->kv_indptr,
                                  batch->kv_indices, batch->rev_input_indptr, batch->positions, batch->rows, stream));
    if (conv_taps > 1 && batch->prefill > 0)
      NF_KERNEL_CHECK(nf_conv_state(kv.dtype, proj, ld, &conv, batch->positions, batch->decode, batch->prefill, stream));
  }
};

// Attention of the decode rows, then of the prompts' portions.
template <class Args, int (*launch)(const Args*, nf_stream_t)>
struct StackPagedAttention : public StackOperator {
  Args args{};
  bool decoding = true, prompts = true;
  const int32_t* page_ids = nullptr;  // pages of another pool than the batch's
  void work() override {
    Args a = args;
    a.input_indptr = batch->input_indptr;
    a.kv_indptr = batch->kv_indptr;
    a.kv_indices = page_ids ? page_ids : batch->kv_indices;
    a.rev_input_indptr = batch->rev_input_indptr;
    a.positions = batch->positions;
    if (batch->decode > 0 && decoding) {
      a.req_begin = 0;
      a.req_num = a.max_rows = batch->decode;
      a.row_begin = 0;
      a.decode = 1;
      NF_KERNEL_CHECK(launch(&a, stream));
    }
    if (batch->prefill > 0 && prompts) {
      a.req_begin = a.row_begin = batch->decode;
      a.req_num = batch->prefill;
      a.max_rows = batch->rows - batch->decode;
      a.decode = 0;
      NF_KERNEL_CHECK(launch(&a, stream));
    }
  }
};
using StackAttention = StackPagedAttention<nf_window_attention_args, nf_window_attention>;
using StackLatentAttention = StackPagedAttention<nf_latent_attention_args, nf_latent_attention>;

struct StackRecurrence : public StackOperator {
  nf_recurrence_args args{};
  void work() override {
    nf_recurrence_args a = args;
    a.input_indptr = batch->input_indptr;
    a.positions = batch->positions;
    a.state_slots = batch->state_slots;
    a.total_rows = batch->rows;
    if (batch->decode > 0) {
      a.req_begin = a.row_begin = 0;
      a.req_num = a.rows = batch->decode;
      NF_KERNEL_CHECK(nf_linear_recurrence(&a, stream));
    }
    if (batch->prefill > 0) {
      a.req_begin = a.row_begin = batch->decode;
      a.req_num = batch->prefill;
      a.rows = batch->rows - batch->decode;
      NF_KERNEL_CHECK(nf_linear_recurrence(&a, stream));
    }
  }
};

// The rows whose logits are wanted, through the model's norm.
struct StackGatherNorm : public StackOperator {
  const float* x = nullptr;
  nf_norm norm{};
  void* out = nullptr;
  int width = 0, ld = 0;
  void work() override {
    NF_KERNEL_CHECK(nf_norm_rows(dtype, x, batch->logit_row_index, &norm, out, batch->logit_rows, width, ld, stream));
  }
};

struct StackArgmax : public StackOperator {
  const float* logits = nullptr;
  int32_t* argmax = nullptr;
  int cols = 0, ld = 0;
  void work() override { NF_KERNEL_CHECK(nf_argmax_f32(logits, argmax, batch->logit_rows, cols, ld, stream)); }
};
