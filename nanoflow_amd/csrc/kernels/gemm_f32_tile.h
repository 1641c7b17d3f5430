#pragma once
// A 64 x 64 output tile of a true 32-bit GEMM on k-contiguous weights, D = act(A . B^T + bias): every product
// and sum in fp32 on v_mfma_f32_16x16x4_f32.
//
// Four wavefronts of 32 x 32.  K slabs of 16 go through registers into LDS rows of 20 floats (16-byte
// aligned, and the 16 rows a fragment read touches fall on different bank groups).
#include "common.h"

namespace nf {

constexpr int kF32Tile = 64, kF32Slab = 16, kF32Pitch = 20;

template <int kAct>
__device__ __forceinline__ float f32_activation(float v) {
  if constexpr (kAct == NF_ACT_SQUARED_RELU) {
    v = fmaxf(v, 0.f);
    return v * v;
  } else if constexpr (kAct == NF_ACT_SILU) {
    return v / (1.f + expf(-v));
  } else if constexpr (kAct == NF_ACT_GELU) {
    return v * (0.5f + 0.5f * erff(v * 0.70710678118654752440f));
  } else {
    return v;
  }
}

// What becomes of a row of the product before it is stored: multiplied by row_scale[m] (null: not); with NF_ACT_GATED the
// columns are pairs of a gate and an up (nf_gated_act) and D has half as many.
struct RowEpilogue {
  const float* row_scale = nullptr;
  float slope = 1.f, shift = 0.f, limit = INFINITY;
};

// The tile at (m0, n0).  Row m of A is row a_rows[m] where a_rows is not null.
template <int kAct>
__device__ __forceinline__ void gemm_f32_tile(const float* __restrict__ A, const float* __restrict__ B, const float* __restrict__ bias,
                                              float* __restrict__ D, int M, int N, int K, int lda, int ldb, int ldd,
                                              const int32_t* __restrict__ a_rows, int m0, int n0,
                                              const RowEpilogue& ep = {}) {
  __shared__ __attribute__((aligned(16))) float sa[kF32Tile * kF32Pitch], sb[kF32Tile * kF32Pitch];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int wm = (wave >> 1) * 32, wn = (wave & 1) * 32, l16 = lane & 15, lq = lane >> 4;
  const int row = threadIdx.x >> 2, kc = (threadIdx.x & 3) * 4;  // the four floats this thread stages of each operand
  const int am = m0 + row < M ? (a_rows ? a_rows[m0 + row] : m0 + row) : -1;
  float4_t acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = float4_t{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < K; k0 += kF32Slab) {
    float4_t a{0.f, 0.f, 0.f, 0.f}, b{0.f, 0.f, 0.f, 0.f};
    if (k0 + kc < K) {  // K is a multiple of 4
      if (am >= 0) a = *reinterpret_cast<const float4_t*>(A + (size_t)am * lda + k0 + kc);
      if (n0 + row < N) b = *reinterpret_cast<const float4_t*>(B + (size_t)(n0 + row) * ldb + k0 + kc);
    }
    __syncthreads();
    *reinterpret_cast<float4_t*>(sa + row * kF32Pitch + kc) = a;
    *reinterpret_cast<float4_t*>(sb + row * kF32Pitch + kc) = b;
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < kF32Slab; kk += 4) {
      float af[2], bf[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        af[i] = sa[(wm + i * 16 + l16) * kF32Pitch + kk + lq];
        bf[i] = sb[(wn + i * 16 + l16) * kF32Pitch + kk + lq];
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(af[i], bf[j], acc[i][j], 0, 0, 0);
    }
  }
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int m = m0 + wm + i * 16 + lq * 4 + r, n = n0 + wn + j * 16 + l16;
        if (kAct == NF_ACT_GATED || ep.row_scale) {
          const float v = acc[i][j][r] * (ep.row_scale && m < M ? ep.row_scale[m] : 1.f);
          if constexpr (kAct == NF_ACT_GATED) {
            const float up = fminf(fmaxf(__shfl_xor(v, 1, 64), -ep.limit), ep.limit), gate = fminf(v, ep.limit);
            if (m < M && n < N && n % 2 == 0) D[(size_t)m * ldd + n / 2] = gate / (1.f + expf(-ep.slope * gate)) * (up + ep.shift);
          } else if (m < M && n < N) {
            D[(size_t)m * ldd + n] = f32_activation<kAct>(v);
          }
          continue;
        }
        if (m < M && n < N) D[(size_t)m * ldd + n] = f32_activation<kAct>(acc[i][j][r] + (bias ? bias[n] : 0.f));
      }
}

}  // namespace nf
