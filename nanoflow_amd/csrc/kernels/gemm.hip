// The fp16 entries of the GEMM family of gemm_impl.h.
#include "gemm_impl.h"

using namespace nf;

// ---- the entry point that allocates nothing: split-K partial sums in a static device array.
// In host code the array's name is only a stand-in for the symbol; its device address is looked
// up once per device (each device holds its own copy) and only that address is handed to kernels.
constexpr size_t kStaticScratchBytes = (size_t)32 << 20;
static __device__ __align__(256) unsigned char scratch[kStaticScratchBytes];
constexpr int kMaxDevices = 64;
static void* g_scratch_ptr[kMaxDevices] = {};  // benign race: every caller stores the same address

static int static_scratch(const char* who, void** out) {
  int dev = -1;
  if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= kMaxDevices) {
    set_error("%s: cannot tell the current device", who);
    return NF_ERR_RUNTIME;
  }
  if (!g_scratch_ptr[dev]) {
    void* p = nullptr;
    const hipError_t e = hipGetSymbolAddress(&p, HIP_SYMBOL(scratch));
    if (e != hipSuccess || !p) {
      set_error("%s: hipGetSymbolAddress(scratch) on device %d: %s", who, dev, hipGetErrorString(e));
      return NF_ERR_RUNTIME;
    }
    g_scratch_ptr[dev] = p;
  }
  *out = g_scratch_ptr[dev];
  return NF_OK;
}

extern "C" {

int nf_gemm_f16(const uint16_t* A, const uint16_t* B, const uint16_t* C, uint16_t* D, int M, int N,
                int K, float alpha, float beta, int b_col_major, nf_stream_t stream) {
  return gemm_entry<F16>("nf_gemm_f16", A, B, C, D, M, N, K, alpha, beta, b_col_major, stream);
}

size_t nf_gemm_workspace_bytes(int M, int N, int K) {
  if (M <= 0 || N <= 0 || K <= 0) return 0;
  int k_per = 0;
  int shares = splitk_plan(M, N, K, &k_per);
  if (shares < 2) shares = dense_split_plan(M, N, K, &k_per);
  return shares < 2 ? 0 : (size_t)shares * M * N * sizeof(float);
}

size_t nf_gemm_workspace_bytes_upto(int max_M, int N, int K) {
  size_t need = 0;
  for (int m = 1; m <= max_M && m <= kSplitMaxRows; ++m) need = std::max(need, nf_gemm_workspace_bytes(m, N, K));
  // above that only the two-share split of launches with few 256 x 256 tiles: every count of tile rows
  for (int m = kSplitMaxRows + 1; m <= max_M; m = (m + 255) / 256 * 256 + 1)
    need = std::max(need, nf_gemm_workspace_bytes(std::min((m + 255) / 256 * 256, max_M), N, K));
  return need;
}

size_t nf_dual_swiglu_workspace_bytes(int M, int N, int K) {
  if (M <= 0 || N <= 0 || K <= 0) return 0;
  int k_per = 0;
  const int shares = splitk_plan_dual(M, N, K, &k_per);
  return shares < 2 ? 0 : (size_t)2 * shares * M * N * sizeof(float);
}

size_t nf_dual_swiglu_workspace_bytes_upto(int max_M, int N, int K) {
  size_t need = 0;
  for (int m = 1; m <= max_M && m <= kTallRows; ++m) need = std::max(need, nf_dual_swiglu_workspace_bytes(m, N, K));
  return need;
}

int nf_dual_swiglu_f16_ws(const uint16_t* A, const uint16_t* Bgate, const uint16_t* Bup, uint16_t* out, int M,
                          int N, int K, int b_col_major, void* workspace, size_t workspace_bytes, nf_stream_t stream) {
  return b_col_major ? dual_ws_entry<F16, true>("nf_dual_swiglu_f16_ws", A, Bgate, Bup, out, M, N, K, workspace,
                                                workspace_bytes, stream)
                     : dual_ws_entry<F16, false>("nf_dual_swiglu_f16_ws", A, Bgate, Bup, out, M, N, K, workspace,
                                                 workspace_bytes, stream);
}

int nf_gemm_f16_ws(const uint16_t* A, const uint16_t* B, const uint16_t* C, uint16_t* D, int M, int N, int K,
                   float alpha, float beta, int b_col_major, void* workspace, size_t workspace_bytes,
                   nf_stream_t stream) {
  return gemm_ws_entry<F16>("nf_gemm_f16_ws", A, B, C, D, M, N, K, alpha, beta, b_col_major, workspace,
                            workspace_bytes, stream);
}

int nf_gemm_f16_noalloc(const uint16_t* A, const uint16_t* B, const uint16_t* C, uint16_t* D, int M, int N, int K,
                        float alpha, float beta, int b_col_major, nf_stream_t stream) {
  // the few-row split only: the two-share split of dense launches is an optimisation that needs more
  // than the array holds at any shape it applies to, and such a launch runs unsplit here
  int k_per = 0;
  const int few = M > 0 && N > 0 && K > 0 ? splitk_plan(M, N, K, &k_per) : 1;
  const size_t need = few < 2 ? 0 : (size_t)few * M * N * sizeof(float);
  NF_REQUIRE(need <= kStaticScratchBytes,
             "nf_gemm_f16_noalloc: %d x %d x %d is split over K through %zu bytes of partial sums; the static "
             "scratch array holds %zu (use nf_gemm_f16_ws with a workspace of your own, or nf_gemm_f16)",
             M, N, K, need, kStaticScratchBytes);
  void* ws = nullptr;
  if (need) {  // shapes that are not split never touch the array
    const int rc = static_scratch("nf_gemm_f16_noalloc", &ws);
    if (rc) return rc;
  }
  return gemm_ws_entry<F16>("nf_gemm_f16_noalloc", A, B, C, D, M, N, K, alpha, beta, b_col_major, ws,
                            need ? kStaticScratchBytes : 0, stream);
}

size_t nf_gemm_noalloc_scratch_bytes(void) { return kStaticScratchBytes; }

int nf_gemm_tile_menu(int index, int* tile_m, int* tile_n, int* k_contiguous_weights_only) {
  if (index >= 0 && index < kTileMenuSize) {
    if (tile_m) *tile_m = kTileMenu[index].bm;
    if (tile_n) *tile_n = kTileMenu[index].bn;
    if (k_contiguous_weights_only) *k_contiguous_weights_only = kTileMenu[index].col_only ? 1 : 0;
  }
  return kTileMenuSize;
}

size_t nf_gemm_tiled_workspace_bytes(int M, int N, int K, int split_k) {
  if (M <= 0 || N <= 0 || K <= 0) return 0;
  int k_per = 0;
  const int shares = forced_shares(K, split_k, &k_per);
  return shares < 2 ? 0 : (size_t)shares * M * N * sizeof(float);
}

int nf_gemm_f16_tiled(const uint16_t* A, const uint16_t* B, const uint16_t* C, uint16_t* D, int M, int N, int K,
                      float alpha, float beta, int b_col_major, int c_is_row, int tile_m, int tile_n, int split_k,
                      void* workspace, size_t workspace_bytes, nf_stream_t stream) {
  const char* who = "nf_gemm_f16_tiled";
  NF_REQUIRE(tile_m > 0 && tile_n > 0, "%s: tile %d x %d", who, tile_m, tile_n);
  int rc = check_gemm_args(who, A, B, D, M, N, K);
  if (rc) return rc;
  NF_REQUIRE(beta == 0.f || C, "%s: beta=%g needs C", who, (double)beta);
  NF_REQUIRE(((uintptr_t)C) % 8 == 0, "%s: C must be 8-byte aligned", who);
  if (M == 0) return NF_OK;
  int k_per = 0;
  const int shares = forced_shares(K, split_k, &k_per);
  NF_REQUIRE(shares < 2 || (workspace && (uintptr_t)workspace % 16 == 0 &&
                            workspace_bytes >= (size_t)shares * M * N * sizeof(float)),
             "%s: a split over K into %d shares needs a 16-byte aligned workspace of %zu bytes (nf_gemm_tiled_workspace_bytes)",
             who, shares, (size_t)shares * M * N * sizeof(float));
  const int index = menu_pick(tile_m, tile_n, b_col_major != 0);
  const int ldc = c_is_row ? 0 : N;
  float* P = static_cast<float*>(workspace);
  hipStream_t s = (hipStream_t)stream;
  return b_col_major ? dispatch_menu<F16, true>(index, A, B, C, D, M, N, K, alpha, beta, ldc, shares, k_per, P, s)
                     : dispatch_menu<F16, false>(index, A, B, C, D, M, N, K, alpha, beta, ldc, shares, k_per, P, s);
}

int nf_gemm_bias_f16_ws(const uint16_t* A, const uint16_t* B, const uint16_t* bias, uint16_t* D, int M, int N,
                        int K, float alpha, float beta, int b_col_major, void* workspace, size_t workspace_bytes,
                        nf_stream_t stream) {
  NF_REQUIRE(bias, "nf_gemm_bias_f16_ws: null bias");
  return gemm_ws_entry<F16>("nf_gemm_bias_f16_ws", A, B, bias, D, M, N, K, alpha, beta, b_col_major, workspace,
                            workspace_bytes, stream, true);
}

int nf_gemm_bias_f16(const uint16_t* A, const uint16_t* B, const uint16_t* bias, uint16_t* D, int M,
                     int N, int K, float alpha, float beta, int b_col_major, nf_stream_t stream) {
  NF_REQUIRE(bias, "nf_gemm_bias_f16: null bias");
  return gemm_entry<F16>("nf_gemm_bias_f16", A, B, bias, D, M, N, K, alpha, beta, b_col_major, stream, true);
}

int nf_dual_swiglu_f16(const uint16_t* A, const uint16_t* Bgate, const uint16_t* Bup, uint16_t* out,
                       int M, int N, int K, int b_col_major, nf_stream_t stream) {
  return b_col_major ? dual_entry<F16, true>("nf_dual_swiglu_f16", A, Bgate, Bup, out, M, N, K, stream)
                     : dual_entry<F16, false>("nf_dual_swiglu_f16", A, Bgate, Bup, out, M, N, K, stream);
}

}  // extern "C"
