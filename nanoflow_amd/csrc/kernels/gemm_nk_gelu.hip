// The GELU form of the k-contiguous bf16 GEMM (a translation unit of its own: the family's
// tiles take a while to compile).
#include "gemm_nk_impl.h"

extern "C" int nf_gemm_nk_gelu_bf16(const uint16_t* A, const uint16_t* B, uint16_t* D, int M, int N, int K,
                                     void* workspace, size_t workspace_bytes, nf_stream_t stream) {
  return gemm_nk_entry<BF16Gelu>("nf_gemm_nk_gelu_bf16", A, B, nullptr, D, M, N, K, workspace, workspace_bytes, stream);
}
