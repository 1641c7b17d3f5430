// True 32-bit GEMM on k-contiguous weights: D = act(A . B^T), every product and sum in fp32 on
// v_mfma_f32_16x16x4_f32.  The projections of a model served in 32-bit; not a throughput kernel.
//
// A workgroup is a 64 x 64 output tile, four wavefronts of 32 x 32.  K slabs of 16 go through
// registers into LDS rows of 20 floats (16-byte aligned, and the 16 rows a fragment read touches
// fall on different bank groups).
#include "common.h"

namespace nf {

constexpr int kTile = 64, kSlab = 16, kPitch = 20;

template <int kAct>
__global__ __launch_bounds__(256) void gemm_nk_f32_kernel(const float* __restrict__ A, const float* __restrict__ B,
                                                          float* __restrict__ D, int M, int N, int K) {
  __shared__ __attribute__((aligned(16))) float sa[kTile * kPitch], sb[kTile * kPitch];
  const int m0 = blockIdx.y * kTile, n0 = blockIdx.x * kTile;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int wm = (wave >> 1) * 32, wn = (wave & 1) * 32, l16 = lane & 15, lq = lane >> 4;
  const int row = threadIdx.x >> 2, kc = (threadIdx.x & 3) * 4;  // the four floats this thread stages of each operand
  float4_t acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = float4_t{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < K; k0 += kSlab) {
    float4_t a{0.f, 0.f, 0.f, 0.f}, b{0.f, 0.f, 0.f, 0.f};
    if (k0 + kc < K) {  // K is a multiple of 4
      if (m0 + row < M) a = *reinterpret_cast<const float4_t*>(A + (size_t)(m0 + row) * K + k0 + kc);
      if (n0 + row < N) b = *reinterpret_cast<const float4_t*>(B + (size_t)(n0 + row) * K + k0 + kc);
    }
    __syncthreads();
    *reinterpret_cast<float4_t*>(sa + row * kPitch + kc) = a;
    *reinterpret_cast<float4_t*>(sb + row * kPitch + kc) = b;
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < kSlab; kk += 4) {
      float af[2], bf[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        af[i] = sa[(wm + i * 16 + l16) * kPitch + kk + lq];
        bf[i] = sb[(wn + i * 16 + l16) * kPitch + kk + lq];
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
        float v = acc[i][j][r];
        if constexpr (kAct == NF_ACT_SQUARED_RELU) {
          v = fmaxf(v, 0.f);
          v *= v;
        }
        if (m < M && n < N) D[(size_t)m * N + n] = v;
      }
}

}  // namespace nf

using namespace nf;

extern "C" int nf_gemm_nk_f32(const float* A, const float* B, float* D, int M, int N, int K, int act,
                              nf_stream_t stream) {
  const char* who = "nf_gemm_nk_f32";
  NF_REQUIRE(M >= 0 && N > 0 && K > 0 && K % 4 == 0, "%s: bad shape M=%d N=%d K=%d (K a multiple of 4)", who, M, N, K);
  NF_REQUIRE(act == NF_ACT_NONE || act == NF_ACT_SQUARED_RELU, "%s: unknown activation %d", who, act);
  if (M == 0) return NF_OK;
  NF_REQUIRE(A && B && D, "%s: null pointer", who);
  NF_REQUIRE(((uintptr_t)A | (uintptr_t)B) % 16 == 0, "%s: operands must be 16-byte aligned", who);
  const dim3 grid((N + kTile - 1) / kTile, (M + kTile - 1) / kTile);
  NF_REQUIRE(grid.y <= 65535, "%s: %d rows exceed the grid", who, M);
  auto kern = act == NF_ACT_SQUARED_RELU ? gemm_nk_f32_kernel<NF_ACT_SQUARED_RELU> : gemm_nk_f32_kernel<NF_ACT_NONE>;
  kern<<<grid, 256, 0, (hipStream_t)stream>>>(A, B, D, M, N, K);
  return check_launch(who);
}
