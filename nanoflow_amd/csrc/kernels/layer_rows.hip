// Row operators of the layer-stack pipeline: embedding plus learned positions, the end of a sublayer (its output,
// normed or put together from experts, added to the residual stream, what a pass over layers starts with, and the next norm), gathered norms,
// gated norm, token shift, token gate, tanh, fp32 argmax.
// HBM-bound; one workgroup per row (token shift: per 1024 columns of a row), 16-byte accesses, the row kept in registers between the
// reduction and the write.  The residual stream is fp32.
#include "layer_common.h"

namespace nf {

constexpr int kRowThreads = 256;
constexpr int kFewRows = 512;
constexpr int kMaxRowVec = 16;  // a row is at most 16 x 256 x 4 = 16384 columns

template <class T>
__global__ __launch_bounds__(kRowThreads) void embed_rows_kernel(const int32_t* __restrict__ tokens,
                                                                 const int32_t* __restrict__ positions,
                                                                 const T* __restrict__ embed, const T* __restrict__ pos, float scale,
                                                                 float* __restrict__ x, T* __restrict__ act, int ld) {
  const int t = blockIdx.x;
  const T* e = embed + (size_t)tokens[t] * ld;
  const T* p = pos ? pos + (size_t)positions[t] * ld : nullptr;
  for (int c = threadIdx.x * 4; c < ld; c += kRowThreads * 4) {
    float4_t v = Act<T>::load4(e + c) * scale;
    if (p) v += Act<T>::load4(p + c);
    *reinterpret_cast<float4_t*>(x + (size_t)t * ld + c) = v;
    if (act) Act<T>::store4(act + (size_t)t * ld + c, v);
  }
}

// A row of up to kVec x kThreads groups of four columns in registers, normed in place; columns from `width` on are zero before and
// after (the vectors are zero there).  `scratch`: 32 floats of LDS no one else uses.
template <int kVec, int kThreads = kRowThreads>
__device__ __forceinline__ void norm_row(float4_t (&v)[kVec], const nf_norm& norm, int width, int ld, float* scratch) {
  const float inv_width = 1.f / (float)width;
  float mean = 0.f;
  if (norm.kind == NF_NORM_LAYER) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < kVec; ++i) s += v[i][0] + v[i][1] + v[i][2] + v[i][3];
    mean = block_sum(s, scratch) * inv_width;
#pragma unroll
    for (int i = 0; i < kVec; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) v[i][e] = (i * kThreads + (int)threadIdx.x) * 4 + e < width ? v[i][e] - mean : 0.f;
  }
  float sq = 0.f;
#pragma unroll
  for (int i = 0; i < kVec; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) sq += v[i][e] * v[i][e];
  const float inv = 1.f / sqrtf(block_sum(sq, scratch + 16) * inv_width + norm.eps);
#pragma unroll
  for (int i = 0; i < kVec; ++i) {
    const int c = (i * kThreads + threadIdx.x) * 4;
    if (c >= ld) continue;
    v[i] = v[i] * inv * *reinterpret_cast<const float4_t*>(norm.weight + c);
    if (norm.bias) v[i] += *reinterpret_cast<const float4_t*>(norm.bias + c);
  }
}

// kVec: 4-column groups per thread, kThreads: of the row, more where there are few rows.  TY: float (summed over `shares` slices) or bf16_t; kMixture: TY rows of experts.
template <class TY, class T, int kVec, bool kMixture, int kThreads>
__global__ __launch_bounds__(kThreads) void residual_rows_kernel(nf_residual_args a, const int32_t* __restrict__ place,
                                                                    const float* __restrict__ weight) {
  __shared__ float scratch[64];
  const int t = blockIdx.x, ld = a.ld;
  const size_t row = (size_t)t * ld, slice = (size_t)a.rows * ld;
  const TY* y = (const TY*)a.y;
  float4_t v[kVec], xr[kVec];
#pragma unroll
  for (int i = 0; i < kVec; ++i) {
    const int c = (i * kThreads + threadIdx.x) * 4;
    v[i] = xr[i] = float4_t{0.f, 0.f, 0.f, 0.f};
    if (c >= ld) continue;
    xr[i] = *reinterpret_cast<const float4_t*>(a.x + row + c);  // in flight together with the sublayer's output
    if constexpr (!kMixture) {
      if (!y) continue;
      if constexpr (std::is_same_v<TY, float>) v[i] = sum_shares(y, slice, row + c, a.shares);
      else v[i] = Act<TY>::load4(y + row + c);
    }
  }
  if constexpr (kMixture) {
    // the token's places and weights, one per lane (at most 64), then row after row by its number
    const int lane = threadIdx.x & 63;
    const int my_place = lane < a.top ? place[(size_t)t * a.top + lane] : -1;
    const float my_weight = lane >= a.top ? 0.f : weight ? weight[(size_t)t * a.top + lane] : 1.f;
    const float same = wave_sum(my_place < 0 ? my_weight : 0.f);  // of identity experts
    float4_t own[kVec];
#pragma unroll
    for (int i = 0; i < kVec; ++i) {
      const int c = (i * kThreads + threadIdx.x) * 4;
      own[i] = same != 0.f && c < ld && a.identity ? Act<TY>::load4((const TY*)a.identity + row + c) : float4_t{0.f, 0.f, 0.f, 0.f};
    }
    constexpr int kAhead = 4;
    for (int k0 = 0; k0 < a.top; k0 += kAhead) {
      float w[kAhead];
      const TY* src[kAhead];
#pragma unroll
      for (int k = 0; k < kAhead; ++k) {
        const int at = k0 + k < a.top ? __builtin_amdgcn_readlane(my_place, k0 + k) : -1;
        w[k] = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(my_weight), min(k0 + k, 63)));
        src[k] = at >= 0 ? y + (size_t)at * a.y_ld : nullptr;
      }
#pragma unroll
      for (int i = 0; i < kVec; ++i) {
        const int c = (i * kThreads + threadIdx.x) * 4;
        if (c >= ld) continue;
        float4_t e[kAhead];
#pragma unroll
        for (int k = 0; k < kAhead; ++k) e[k] = src[k] ? Act<TY>::load4(src[k] + c) : float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < kAhead; ++k) v[i] += e[k] * w[k];
      }
    }
#pragma unroll
    for (int i = 0; i < kVec; ++i) v[i] += own[i] * same;
  }
  if (a.y_norm.kind != NF_NORM_NONE) norm_row<kVec, kThreads>(v, a.y_norm, a.width, ld, scratch);
  const T* e = a.table ? (const T*)a.table + (size_t)a.tokens[t] * ld : nullptr;
#pragma unroll
  for (int i = 0; i < kVec; ++i) {
    const int c = (i * kThreads + threadIdx.x) * 4;
    v[i] = v[i] * a.y_scale + xr[i];
    if (e && c < ld) v[i] += Act<T>::load4(e + c) * a.table_scale;
    if (a.add && c < ld) v[i] += *reinterpret_cast<const float4_t*>(a.add + c);
    if (c < ld) *reinterpret_cast<float4_t*>(a.x + row + c) = v[i];
  }
  if (!a.act) return;
  if (a.next.kind != NF_NORM_NONE) norm_row<kVec, kThreads>(v, a.next, a.width, ld, scratch + 32);
#pragma unroll
  for (int i = 0; i < kVec; ++i) {
    const int c = (i * kThreads + threadIdx.x) * 4;
    if (c < ld) Act<T>::store4((T*)a.act + row + c, v[i]);
  }
}

template <class T, int kVec>
__global__ __launch_bounds__(kRowThreads) void norm_rows_kernel(const float* __restrict__ x, const int32_t* __restrict__ row_index,
                                                                nf_norm norm, T* __restrict__ out, int width, int ld) {
  __shared__ float scratch[32];
  const size_t row = (size_t)(row_index ? row_index[blockIdx.x] : (int)blockIdx.x) * ld;
  float4_t v[kVec];
#pragma unroll
  for (int i = 0; i < kVec; ++i) {
    const int c = (i * kRowThreads + threadIdx.x) * 4;
    v[i] = c < ld ? *reinterpret_cast<const float4_t*>(x + row + c) : float4_t{0.f, 0.f, 0.f, 0.f};
  }
  norm_row<kVec>(v, norm, width, ld, scratch);
#pragma unroll
  for (int i = 0; i < kVec; ++i) {
    const int c = (i * kRowThreads + threadIdx.x) * 4;
    if (c < ld) Act<T>::store4(out + (size_t)blockIdx.x * ld + c, v[i]);
  }
}

// RMS norm of a row, times sigmoid(g), in place.
template <class T, int kVec>
__global__ __launch_bounds__(kRowThreads) void gated_norm_rows_kernel(T* __restrict__ o, int o_ld, const T* __restrict__ g, int g_ld,
                                                                      const float* __restrict__ weight, int width, float eps) {
  __shared__ float scratch[32];
  o += (size_t)blockIdx.x * o_ld;
  g += (size_t)blockIdx.x * g_ld;
  const bool four = (o_ld | g_ld) % 4 == 0;  // rows start at four-element groups
  float4_t v[kVec], gate[kVec];
  auto load = [&](const T* p, int c) {
    float4_t r{0.f, 0.f, 0.f, 0.f};
    if (four && c + 4 <= width) return Act<T>::load4(p + c);
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (c + e < width) r[e] = Act<T>::load(p + c + e);
    return r;
  };
#pragma unroll
  for (int i = 0; i < kVec; ++i) {
    const int c = (i * kRowThreads + threadIdx.x) * 4;
    v[i] = load(o, c);
    gate[i] = load(g, c);
  }
  norm_row<kVec>(v, nf_norm{NF_NORM_RMS, weight, nullptr, eps}, width, (width + 3) / 4 * 4, scratch);
#pragma unroll
  for (int i = 0; i < kVec; ++i) {
    const int c = (i * kRowThreads + threadIdx.x) * 4;
#pragma unroll
    for (int e = 0; e < 4; ++e) v[i][e] *= sigmoid<T>(gate[i][e]);
    if (four && c + 4 <= width) {
      Act<T>::store4(o + c, v[i]);
      continue;
    }
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (c + e < width) Act<T>::store(o + c + e, v[i][e]);
  }
}

template <class T>
__global__ __launch_bounds__(256) void token_gate_rows_kernel(const float* __restrict__ sums, int shares,
                                                              const int32_t* __restrict__ tokens, const T* __restrict__ table,
                                                              int table_ld, int col0, int dim, T* __restrict__ out, int cols, size_t groups) {
  const size_t g = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (g >= groups) return;
  const int t = (int)(g * 4 / cols), c = (int)(g * 4 % cols);
  float4_t v = sum_shares(sums, groups * 4, g * 4, shares);
  const T* e = table + (size_t)tokens[t] * table_ld + col0;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float z = v[i], u = 0.79788456080286535588f * (z + 0.044715f * z * z * z);
    v[i] = c + i < dim ? 0.5f * z * (1.f + tanhf(u)) * Act<T>::load(e + c + i) : 0.f;
  }
  Act<T>::store4(out + g * 4, v);
}

template <class T>
__global__ __launch_bounds__(kRowThreads) void token_shift_kernel(
    const float* __restrict__ x, const float* __restrict__ shift_state, const float* __restrict__ mu, T* __restrict__ out,
    int n_mix, const int32_t* __restrict__ input_indptr, const int32_t* __restrict__ rev_input_indptr,
    const int32_t* __restrict__ positions, const int32_t* __restrict__ state_slots, int rows, int ld) {
  const int t = blockIdx.x, req = rev_input_indptr[t];
  const float* prev = nullptr;  // the token before this one: a row of the batch, the state, or nothing
  if (positions[t] > 0) prev = t > input_indptr[req] ? x + (size_t)(t - 1) * ld : shift_state + (size_t)state_slots[req] * ld;
  const int c = (blockIdx.y * kRowThreads + threadIdx.x) * 4;
  if (c < ld) {
    const float4_t h = *reinterpret_cast<const float4_t*>(x + (size_t)t * ld + c);
    const float4_t p = prev ? *reinterpret_cast<const float4_t*>(prev + c) : float4_t{0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < n_mix; ++s) {
      const float4_t m = *reinterpret_cast<const float4_t*>(mu + (size_t)s * ld + c);
      Act<T>::store4(out + ((size_t)s * rows + t) * ld + c, h + (p - h) * m);
    }
  }
}

template <class T>
__global__ __launch_bounds__(256) void tanh_rows_kernel(const float* __restrict__ sums, int shares, T* __restrict__ out,
                                                        size_t groups) {
  const size_t g = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (g >= groups) return;
  float4_t v = sum_shares(sums, groups * 4, g * 4, shares);
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = tanhf(v[e]);
  Act<T>::store4(out + g * 4, v);
}

__global__ __launch_bounds__(1024) void argmax_f32_kernel(const float* __restrict__ logits, int32_t* __restrict__ argmax,
                                                          int cols, int ld) {
  __shared__ float s_val[16];
  __shared__ int s_idx[16];
  const float* row = logits + (size_t)blockIdx.x * ld;
  float best = -INFINITY;
  int at = 0x7fffffff;
  auto take = [&](float v, int i) {
    if (v > best || (v == best && i < at)) {
      best = v;
      at = i;
    }
  };
  for (int c = threadIdx.x; c < cols; c += 1024) take(row[c], c);
#pragma unroll
  for (int m = 32; m > 0; m >>= 1) {
    const float v = __shfl_xor(best, m, 64);
    const int i = __shfl_xor(at, m, 64);
    take(v, i);
  }
  if ((threadIdx.x & 63) == 0) {
    s_val[threadIdx.x >> 6] = best;
    s_idx[threadIdx.x >> 6] = at;
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < 16; ++w) take(s_val[w], s_idx[w]);
    argmax[blockIdx.x] = at < cols ? at : 0;  // a row without a number in it (all NaN) gives column 0
  }
}

template <class F>
static int with_vec(int ld, F&& f) {
  const int vec = (ld / 4 + kRowThreads - 1) / kRowThreads;
  if (vec <= 1) return f(ic<1>{});
  if (vec <= 2) return f(ic<2>{});
  if (vec <= 4) return f(ic<4>{});
  if (vec <= 8) return f(ic<8>{});
  return f(ic<16>{});
}

}  // namespace nf

using namespace nf;

static int check_rows(const char* who, int dtype, int rows, int width, int ld) {
  NF_REQUIRE(dtype == NF_F32 || dtype == NF_BF16, "%s: unknown dtype %d", who, dtype);
  NF_REQUIRE(rows >= 0 && width > 0 && ld >= width && ld % 8 == 0 && ld <= kMaxRowVec * kRowThreads * 4,
             "%s: rows=%d width=%d ld=%d (ld a multiple of 8, at most %d)", who, rows, width, ld,
             kMaxRowVec * kRowThreads * 4);
  return NF_OK;
}

static int check_norm(const char* who, const nf_norm& n) {
  NF_REQUIRE(n.kind == NF_NORM_NONE || n.kind == NF_NORM_RMS || n.kind == NF_NORM_LAYER, "%s: unknown norm %d", who, n.kind);
  NF_REQUIRE(n.kind == NF_NORM_NONE || n.weight, "%s: a norm without a weight", who);
  return NF_OK;
}

extern "C" {

int nf_embed_rows(int dtype, const int32_t* tokens, const int32_t* positions, const void* embed, const void* pos, float scale, float* x,
                  void* act, int rows, int ld, nf_stream_t stream) {
  int rc = check_rows("nf_embed_rows", dtype, rows, 1, ld);
  if (rc) return rc;
  if (rows == 0) return NF_OK;
  NF_REQUIRE(tokens && embed && x && (!pos || positions), "nf_embed_rows: null pointer");
  hipStream_t s = (hipStream_t)stream;
  if (dtype == NF_BF16)
    embed_rows_kernel<bf16_t><<<rows, kRowThreads, 0, s>>>(tokens, positions, (const bf16_t*)embed, (const bf16_t*)pos, scale, x,
                                                           (bf16_t*)act, ld);
  else
    embed_rows_kernel<float><<<rows, kRowThreads, 0, s>>>(tokens, positions, (const float*)embed, (const float*)pos, scale, x,
                                                          (float*)act, ld);
  return check_launch("nf_embed_rows");
}

int nf_residual_rows(const nf_residual_args* args, nf_stream_t stream) {
  const char* who = "nf_residual_rows";
  NF_REQUIRE(args, "%s: null pointer", who);
  const nf_residual_args& a = *args;
  int rc = check_rows(who, a.dtype, a.rows, a.width, a.ld);
  if (rc || (rc = check_norm(who, a.y_norm)) || (rc = check_norm(who, a.next))) return rc;
  if (a.routing) {
    NF_REQUIRE(a.top >= 1 && a.top <= 64 && a.y_ld >= a.ld && a.y_ld % 4 == 0 && a.routing->place && (a.routing->weight || !a.identity),
               "%s: incomplete routing (top %d, stride %d)", who, a.top, a.y_ld);
  } else if (a.y || a.shares != 0) {
    NF_REQUIRE((a.y_dtype == NF_F32 && a.shares >= 1 && a.shares <= kMaxShares) || (a.y_dtype == NF_BF16 && a.shares == 1),
               "%s: %d shares of dtype %d", who, a.shares, a.y_dtype);
  }
  if (a.rows == 0) return NF_OK;
  NF_REQUIRE((a.y || (!a.routing && a.y_norm.kind == NF_NORM_NONE)) && a.x && (!a.table || a.tokens), "%s: null pointer", who);
  hipStream_t s = (hipStream_t)stream;
  auto sized = [&](auto vec, auto threads) {
    constexpr int V = decltype(vec)::value, N = decltype(threads)::value;
    auto go = [&](auto kern) {
      kern<<<a.rows, N, 0, s>>>(a, a.routing ? a.routing->place : nullptr, a.routing ? a.routing->weight : nullptr);
      return check_launch(who);
    };
    const bool b16 = a.dtype == NF_BF16;
    if (a.routing) return b16 ? go(residual_rows_kernel<bf16_t, bf16_t, V, true, N>) : go(residual_rows_kernel<float, float, V, true, N>);
    if (a.y && a.y_dtype == NF_BF16) return b16 ? go(residual_rows_kernel<bf16_t, bf16_t, V, false, N>) : go(residual_rows_kernel<bf16_t, float, V, false, N>);
    return b16 ? go(residual_rows_kernel<float, bf16_t, V, false, N>) : go(residual_rows_kernel<float, float, V, false, N>);
  };
  // a row on more wavefronts where rows alone leave the CUs mostly empty, and where it is put together from many
  if ((a.rows <= kFewRows || a.routing) && a.ld > 1024) return a.ld <= 4096 ? sized(ic<1>{}, ic<1024>{}) : a.ld <= 8192 ? sized(ic<2>{}, ic<1024>{}) : sized(ic<4>{}, ic<1024>{});
  return with_vec(a.ld, [&](auto v) { return sized(v, ic<kRowThreads>{}); });
}

int nf_norm_rows(int dtype, const float* x, const int32_t* row_index, const nf_norm* norm, void* out, int n, int width, int ld,
                 nf_stream_t stream) {
  int rc = check_rows("nf_norm_rows", dtype, n, width, ld);
  if (rc) return rc;
  NF_REQUIRE(norm && norm->kind != NF_NORM_NONE, "nf_norm_rows: no norm");
  if ((rc = check_norm("nf_norm_rows", *norm))) return rc;
  if (n == 0) return NF_OK;
  NF_REQUIRE(x && out, "nf_norm_rows: null pointer");
  hipStream_t s = (hipStream_t)stream;
  return with_vec(ld, [&](auto v) {
    constexpr int V = decltype(v)::value;
    if (dtype == NF_BF16) norm_rows_kernel<bf16_t, V><<<n, kRowThreads, 0, s>>>(x, row_index, *norm, (bf16_t*)out, width, ld);
    else norm_rows_kernel<float, V><<<n, kRowThreads, 0, s>>>(x, row_index, *norm, (float*)out, width, ld);
    return check_launch("nf_norm_rows");
  });
}

int nf_gated_norm_rows(int dtype, void* o, int o_ld, const void* g, int g_ld, const float* weight, int rows, int width, float eps,
                       nf_stream_t stream) {
  const char* who = "nf_gated_norm_rows";
  int rc = check_rows(who, dtype, rows, width, (width + 7) / 8 * 8);
  if (rc) return rc;
  NF_REQUIRE(o_ld >= width && g_ld >= width, "%s: strides %d, %d below %d columns", who, o_ld, g_ld, width);
  if (rows == 0) return NF_OK;
  NF_REQUIRE(o && g && weight, "%s: null pointer", who);
  NF_REQUIRE(((uintptr_t)o | (uintptr_t)g) % (dtype == NF_BF16 ? 8 : 16) == 0, "%s: rows must start at groups of four", who);
  hipStream_t s = (hipStream_t)stream;
  return with_vec(width + 3, [&](auto v) {
    constexpr int V = decltype(v)::value;
    if (dtype == NF_BF16) gated_norm_rows_kernel<bf16_t, V><<<rows, kRowThreads, 0, s>>>((bf16_t*)o, o_ld, (const bf16_t*)g, g_ld, weight, width, eps);
    else gated_norm_rows_kernel<float, V><<<rows, kRowThreads, 0, s>>>((float*)o, o_ld, (const float*)g, g_ld, weight, width, eps);
    return check_launch(who);
  });
}

int nf_token_gate_rows(int dtype, const float* sums, int shares, const int32_t* tokens, const void* table, int table_ld, int col0, int dim,
                       void* out, int rows, int cols, nf_stream_t stream) {
  const char* who = "nf_token_gate_rows";
  NF_REQUIRE(dtype == NF_F32 || dtype == NF_BF16, "%s: unknown dtype %d", who, dtype);
  NF_REQUIRE(rows >= 0 && cols > 0 && cols % 4 == 0 && dim > 0 && dim <= cols && shares >= 1 && shares <= kMaxShares && col0 >= 0 &&
                 col0 + dim <= table_ld,
             "%s: rows=%d cols=%d dim=%d shares=%d, table columns %d + %d of %d", who, rows, cols, dim, shares, col0, dim, table_ld);
  if (rows == 0) return NF_OK;
  NF_REQUIRE(sums && tokens && table && out, "%s: null pointer", who);
  const size_t groups = (size_t)rows * cols / 4;
  const unsigned grid = (unsigned)((groups + 255) / 256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == NF_BF16)
    token_gate_rows_kernel<bf16_t><<<grid, 256, 0, s>>>(sums, shares, tokens, (const bf16_t*)table, table_ld, col0, dim, (bf16_t*)out, cols, groups);
  else
    token_gate_rows_kernel<float><<<grid, 256, 0, s>>>(sums, shares, tokens, (const float*)table, table_ld, col0, dim, (float*)out, cols, groups);
  return check_launch(who);
}

int nf_token_shift(int dtype, const float* x, const float* shift_state, const float* mu, void* out, int n_mix,
                   const int32_t* input_indptr, const int32_t* rev_input_indptr, const int32_t* positions,
                   const int32_t* state_slots, int rows, int ld, nf_stream_t stream) {
  int rc = check_rows("nf_token_shift", dtype, rows, 1, ld);
  if (rc) return rc;
  NF_REQUIRE(n_mix >= 1 && n_mix <= 16, "nf_token_shift: %d mixes", n_mix);
  if (rows == 0) return NF_OK;
  NF_REQUIRE(x && shift_state && mu && out && input_indptr && rev_input_indptr && positions && state_slots,
             "nf_token_shift: null pointer");
  hipStream_t s = (hipStream_t)stream;
  const dim3 grid((unsigned)rows, (unsigned)((ld / 4 + kRowThreads - 1) / kRowThreads));
  if (dtype == NF_BF16)
    token_shift_kernel<bf16_t><<<grid, kRowThreads, 0, s>>>(x, shift_state, mu, (bf16_t*)out, n_mix, input_indptr,
                                                            rev_input_indptr, positions, state_slots, rows, ld);
  else
    token_shift_kernel<float><<<grid, kRowThreads, 0, s>>>(x, shift_state, mu, (float*)out, n_mix, input_indptr,
                                                           rev_input_indptr, positions, state_slots, rows, ld);
  return check_launch("nf_token_shift");
}

int nf_tanh_rows(int dtype, const float* sums, int shares, void* out, int rows, int cols, nf_stream_t stream) {
  NF_REQUIRE(dtype == NF_F32 || dtype == NF_BF16, "nf_tanh_rows: unknown dtype %d", dtype);
  NF_REQUIRE(rows >= 0 && cols > 0 && cols % 4 == 0 && shares >= 1 && shares <= kMaxShares,
             "nf_tanh_rows: rows=%d cols=%d shares=%d", rows, cols, shares);
  if (rows == 0) return NF_OK;
  NF_REQUIRE(sums && out, "nf_tanh_rows: null pointer");
  const size_t groups = (size_t)rows * cols / 4;
  const unsigned grid = (unsigned)((groups + 255) / 256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == NF_BF16) tanh_rows_kernel<bf16_t><<<grid, 256, 0, s>>>(sums, shares, (bf16_t*)out, groups);
  else tanh_rows_kernel<float><<<grid, 256, 0, s>>>(sums, shares, (float*)out, groups);
  return check_launch("nf_tanh_rows");
}

int nf_argmax_f32(const float* logits, int32_t* argmax, int rows, int cols, int ld, nf_stream_t stream) {
  NF_REQUIRE(rows >= 0 && cols > 0 && ld >= cols, "nf_argmax_f32: rows=%d cols=%d ld=%d", rows, cols, ld);
  if (rows == 0) return NF_OK;
  NF_REQUIRE(logits && argmax, "nf_argmax_f32: null pointer");
  argmax_f32_kernel<<<rows, 1024, 0, (hipStream_t)stream>>>(logits, argmax, cols, ld);
  return check_launch("nf_argmax_f32");
}

}  // extern "C"
