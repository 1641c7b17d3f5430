// Row operators of the layer-stack pipeline: embedding plus learned positions, norm of a sublayer's
// output added to the residual stream, token shift, tanh, the gathered final norm, fp32 argmax.
// HBM-bound; one workgroup per row (token shift: per 1024 columns of a row), 16-byte accesses, the row kept in registers between the
// reduction and the write.  The residual stream is fp32.
#include "layer_common.h"

namespace nf {

constexpr int kRowThreads = 256;
constexpr int kMaxRowVec = 16;  // a row is at most 16 x 256 x 4 = 16384 columns

template <class T>
__global__ __launch_bounds__(kRowThreads) void embed_rows_kernel(const int32_t* __restrict__ tokens,
                                                                 const int32_t* __restrict__ positions,
                                                                 const T* __restrict__ embed, const T* __restrict__ pos,
                                                                 float* __restrict__ x, T* __restrict__ act, int ld) {
  const int t = blockIdx.x;
  const T* e = embed + (size_t)tokens[t] * ld;
  const T* p = pos ? pos + (size_t)positions[t] * ld : nullptr;
  for (int c = threadIdx.x * 4; c < ld; c += kRowThreads * 4) {
    float4_t v = Act<T>::load4(e + c);
    if (p) v += Act<T>::load4(p + c);
    *reinterpret_cast<float4_t*>(x + (size_t)t * ld + c) = v;
    if (act) Act<T>::store4(act + (size_t)t * ld + c, v);
  }
}

// kVec: 4-column groups per thread.  TY: float (summed over `shares` slices) or bf16_t.
template <class TY, class T, int kVec>
__global__ __launch_bounds__(kRowThreads) void norm_add_rows_kernel(const TY* __restrict__ y, int shares,
                                                                    const float* __restrict__ weight, float* __restrict__ x,
                                                                    T* __restrict__ act, int rows, float inv_width, int ld,
                                                                    float eps) {
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  const size_t row = (size_t)t * ld, slice = (size_t)rows * ld;
  float4_t v[kVec], xr[kVec];
  float sq = 0.f;
#pragma unroll
  for (int i = 0; i < kVec; ++i) {
    const int c = (i * kRowThreads + threadIdx.x) * 4;
    v[i] = float4_t{0.f, 0.f, 0.f, 0.f};
    if (c < ld) {
      xr[i] = *reinterpret_cast<const float4_t*>(x + row + c);  // in flight together with the sublayer's output
      if constexpr (std::is_same_v<TY, float>) v[i] = sum_shares(y, slice, row + c, shares);
      else v[i] = Act<TY>::load4(y + row + c);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) sq += v[i][e] * v[i][e];
  }
  const float inv = 1.f / sqrtf(block_sum(sq, scratch) * inv_width + eps);
#pragma unroll
  for (int i = 0; i < kVec; ++i) {
    const int c = (i * kRowThreads + threadIdx.x) * 4;
    if (c >= ld) continue;
    const float4_t r = xr[i] + v[i] * inv * *reinterpret_cast<const float4_t*>(weight + c);
    *reinterpret_cast<float4_t*>(x + row + c) = r;
    if (act) Act<T>::store4(act + row + c, r);
  }
}

template <class T, int kVec>
__global__ __launch_bounds__(kRowThreads) void gather_norm_rows_kernel(const float* __restrict__ x,
                                                                       const int32_t* __restrict__ row_index,
                                                                       const float* __restrict__ weight,
                                                                       T* __restrict__ out, float inv_width, int ld, float eps) {
  __shared__ float scratch[16];
  const size_t row = (size_t)row_index[blockIdx.x] * ld;
  float4_t v[kVec];
  float sq = 0.f;
#pragma unroll
  for (int i = 0; i < kVec; ++i) {
    const int c = (i * kRowThreads + threadIdx.x) * 4;
    v[i] = c < ld ? *reinterpret_cast<const float4_t*>(x + row + c) : float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) sq += v[i][e] * v[i][e];
  }
  const float inv = 1.f / sqrtf(block_sum(sq, scratch) * inv_width + eps);
#pragma unroll
  for (int i = 0; i < kVec; ++i) {
    const int c = (i * kRowThreads + threadIdx.x) * 4;
    if (c < ld) Act<T>::store4(out + (size_t)blockIdx.x * ld + c, v[i] * inv * *reinterpret_cast<const float4_t*>(weight + c));
  }
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

extern "C" {

int nf_embed_rows(int dtype, const int32_t* tokens, const int32_t* positions, const void* embed, const void* pos, float* x,
                  void* act, int rows, int ld, nf_stream_t stream) {
  int rc = check_rows("nf_embed_rows", dtype, rows, 1, ld);
  if (rc) return rc;
  if (rows == 0) return NF_OK;
  NF_REQUIRE(tokens && embed && x && (!pos || positions), "nf_embed_rows: null pointer");
  hipStream_t s = (hipStream_t)stream;
  if (dtype == NF_BF16)
    embed_rows_kernel<bf16_t><<<rows, kRowThreads, 0, s>>>(tokens, positions, (const bf16_t*)embed, (const bf16_t*)pos, x,
                                                           (bf16_t*)act, ld);
  else
    embed_rows_kernel<float><<<rows, kRowThreads, 0, s>>>(tokens, positions, (const float*)embed, (const float*)pos, x,
                                                          (float*)act, ld);
  return check_launch("nf_embed_rows");
}

int nf_norm_add_rows(int y_dtype, const void* y, int shares, const float* weight, float* x, int dtype, void* act, int rows,
                     int width, int ld, float eps, nf_stream_t stream) {
  int rc = check_rows("nf_norm_add_rows", dtype, rows, width, ld);
  if (rc) return rc;
  NF_REQUIRE((y_dtype == NF_F32 && shares >= 1 && shares <= kMaxShares) || (y_dtype == NF_BF16 && shares == 1),
             "nf_norm_add_rows: %d shares of dtype %d", shares, y_dtype);
  if (rows == 0) return NF_OK;
  NF_REQUIRE(y && weight && x, "nf_norm_add_rows: null pointer");
  hipStream_t s = (hipStream_t)stream;
  const float inv = 1.0f / (float)width;
  return with_vec(ld, [&](auto v) {
    constexpr int V = decltype(v)::value;
    if (y_dtype == NF_BF16 && dtype == NF_BF16)
      norm_add_rows_kernel<bf16_t, bf16_t, V><<<rows, kRowThreads, 0, s>>>((const bf16_t*)y, shares, weight, x, (bf16_t*)act,
                                                                           rows, inv, ld, eps);
    else if (y_dtype == NF_BF16)
      norm_add_rows_kernel<bf16_t, float, V><<<rows, kRowThreads, 0, s>>>((const bf16_t*)y, shares, weight, x, (float*)act,
                                                                          rows, inv, ld, eps);
    else if (dtype == NF_BF16)
      norm_add_rows_kernel<float, bf16_t, V><<<rows, kRowThreads, 0, s>>>((const float*)y, shares, weight, x, (bf16_t*)act,
                                                                          rows, inv, ld, eps);
    else
      norm_add_rows_kernel<float, float, V><<<rows, kRowThreads, 0, s>>>((const float*)y, shares, weight, x, (float*)act,
                                                                         rows, inv, ld, eps);
    return check_launch("nf_norm_add_rows");
  });
}

int nf_gather_norm_rows(int dtype, const float* x, const int32_t* row_index, const float* weight, void* out, int n, int width,
                        int ld, float eps, nf_stream_t stream) {
  int rc = check_rows("nf_gather_norm_rows", dtype, n, width, ld);
  if (rc) return rc;
  if (n == 0) return NF_OK;
  NF_REQUIRE(x && row_index && weight && out, "nf_gather_norm_rows: null pointer");
  hipStream_t s = (hipStream_t)stream;
  return with_vec(ld, [&](auto v) {
    constexpr int V = decltype(v)::value;
    if (dtype == NF_BF16)
      gather_norm_rows_kernel<bf16_t, V><<<n, kRowThreads, 0, s>>>(x, row_index, weight, (bf16_t*)out, 1.0f / width, ld, eps);
    else
      gather_norm_rows_kernel<float, V><<<n, kRowThreads, 0, s>>>(x, row_index, weight, (float*)out, 1.0f / width, ld, eps);
    return check_launch("nf_gather_norm_rows");
  });
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
