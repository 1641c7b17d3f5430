// The bf16 entries of the GEMM family that take weights in either layout, and the bf16 gate/up pair.
#include "gemm_impl.h"

extern "C" {

int nf_gemm_bf16(const uint16_t* A, const uint16_t* B, const uint16_t* C, uint16_t* D, int M, int N,
                 int K, float alpha, float beta, int b_col_major, nf_stream_t stream) {
  return gemm_entry<BF16>("nf_gemm_bf16", A, B, C, D, M, N, K, alpha, beta, b_col_major, stream);
}

int nf_dual_swiglu_bf16(const uint16_t* A, const uint16_t* Bgate, const uint16_t* Bup, uint16_t* out,
                        int M, int N, int K, nf_stream_t stream) {
  return dual_entry<BF16, false>("nf_dual_swiglu_bf16", A, Bgate, Bup, out, M, N, K, stream);
}

}  // extern "C"
