// Grouped GEMMs on k-contiguous weights, D_g = act(A_g . B_g^T): the experts of a mixture (every group has the
// rows its router chose, found through the routing's tile list and gathered while they are loaded) and
// per-head products (every group has all rows and columns of its own).
//
// bf16: the tiles of the plain GEMM family; an m tile never spans two groups.  fp32: gemm_f32's tile.
#include "gemm_f32_tile.h"
#include "gemm_impl.h"

namespace {

struct TilePlace {
  int group, m_base, rows, n_tile;  // rows: of the group
  size_t row0;                      // the group's first row in A (routed, not gathered) and in D
};

// Tile `logical` of the launch; group -1: past the end.  Inside a routed group the m tiles are fastest: they run side by
// side and share a panel of the expert's weights, which is read once.
template <int BM>
__device__ __forceinline__ TilePlace find_tile(const nf_grouped_gemm_args& a, int bid, int tiles_n) {
  const int tiles_m = (a.M + BM - 1) / BM;
  const int m_tiles = a.routing.n_tiles ? *a.routing.n_tiles : tiles_m * a.groups;
  const int total = m_tiles * tiles_n, logical = xcd_order(bid, total);
  if (bid / 8 >= (total + 7) / 8 || logical >= total) return {-1, 0, 0, 0, 0};
  const int mt = logical / tiles_n, n_tile = logical % tiles_n;
  if (a.routing.n_tiles) {
    const int g = a.routing.tile_group[mt], first = a.routing.offsets[g], rows = a.routing.offsets[g + 1] - first;
    const int i = logical - (mt - a.routing.tile_row[mt] / BM) * tiles_n, tiles = (rows + BM - 1) / BM;
    return {g, i % tiles * BM, rows, i / tiles, (size_t)first};
  }
  return {mt / tiles_m, mt % tiles_m * BM, a.M, n_tile, 0};
}

template <class E, int BM, int BN, int WM, int WN>
__global__ __launch_bounds__(WM * WN * 64) void gemm_grouped_kernel(nf_grouped_gemm_args a, int tiles_n) {
  const TilePlace t = find_tile<BM>(a, blockIdx.x, tiles_n);
  if (t.group < 0) return;
  const bool routed = a.routing.n_tiles != nullptr;
  const int32_t* rows = routed && a.gather ? a.routing.row_of + t.row0 : nullptr;
  const uint16_t* A = (const uint16_t*)a.a + (routed ? (rows ? 0 : t.row0 * a.lda) : (size_t)t.group * a.a_group);
  uint16_t* D = (uint16_t*)a.d + (routed ? t.row0 * a.ldd : (size_t)t.group * a.d_group);
  GroupEpilogue ep;
  if (routed && a.weigh) ep.row_scale = a.routing.row_weight + t.row0;
  if constexpr (std::is_same_v<E, BF16Gated>) {
    ep.slope = a.gated.slope;
    ep.shift = a.gated.shift;
    if (a.gated.limits) ep.limit = a.gated.limits[t.group];
  }
  gemm_tile<E, BM, BN, WM, WN, false, true, false, true>(A, (const uint16_t*)a.b + (size_t)t.group * a.N * a.K, nullptr, nullptr, D,
                                                         t.rows, a.N, a.K, 1.f, 0.f, a.N, t.m_base, t.n_tile * BN, a.lda, a.K, a.ldd,
                                                         rows, a.M, ep);
}

template <int kAct>
__global__ __launch_bounds__(256) void gemm_grouped_f32_kernel(nf_grouped_gemm_args a, int tiles_n) {
  const TilePlace t = find_tile<kF32Tile>(a, blockIdx.x, tiles_n);
  if (t.group < 0) return;
  const bool routed = a.routing.n_tiles != nullptr;
  const int32_t* rows = routed && a.gather ? a.routing.row_of + t.row0 : nullptr;
  const float* A = (const float*)a.a + (routed ? (rows ? 0 : t.row0 * a.lda) : (size_t)t.group * a.a_group);
  float* D = (float*)a.d + (routed ? t.row0 * a.ldd : (size_t)t.group * a.d_group);
  RowEpilogue ep;
  if (routed && a.weigh) ep.row_scale = a.routing.row_weight + t.row0;
  if constexpr (kAct == NF_ACT_GATED) {
    ep.slope = a.gated.slope;
    ep.shift = a.gated.shift;
    if (a.gated.limits) ep.limit = a.gated.limits[t.group];
  }
  gemm_f32_tile<kAct>(A, (const float*)a.b + (size_t)t.group * a.N * a.K, nullptr, D, t.rows, a.N, a.K, a.lda, a.K, a.ldd, rows, t.m_base,
                      t.n_tile * kF32Tile, ep);
}

unsigned grid_of(const nf_grouped_gemm_args& a, int bm, int tiles_n) {
  const long long m_tiles = a.routing.n_tiles ? (long long)a.max_rows / bm + std::min(a.groups, a.max_rows) : (long long)((a.M + bm - 1) / bm) * a.groups;
  return (unsigned)((m_tiles * tiles_n + 7) / 8 * 8);
}

template <class E, int BM, int BN, int WM, int WN>
int launch_grouped(const nf_grouped_gemm_args& a, hipStream_t s) {
  using SM = GemmSmem<BM, BN, 1>;
  auto kern = gemm_grouped_kernel<E, BM, BN, WM, WN>;
  static bool attr_set = false;  // benign race: the call is idempotent
  if (!attr_set) {
    const hipError_t e =
        hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)SM::bytes);
    if (e != hipSuccess) {
      set_error("nf_gemm_grouped: cannot reserve %zu bytes of LDS: %s", SM::bytes, hipGetErrorString(e));
      return NF_ERR_RUNTIME;
    }
    attr_set = true;
  }
  const int tiles_n = (a.N + BN - 1) / BN;
  kern<<<grid_of(a, BM, tiles_n), WM * WN * 64, SM::bytes, s>>>(a, tiles_n);
  return check_launch("nf_gemm_grouped");
}

template <class E>
int dispatch_grouped(const nf_grouped_gemm_args& a, int tile_rows, hipStream_t s) {
  if (tile_rows == 64) return a.N <= 128 ? launch_grouped<E, 64, 128, 2, 2>(a, s) : launch_grouped<E, 64, 256, 1, 4>(a, s);
  return a.N > 128 && a.N % 256 == 0 ? launch_grouped<E, 128, 256, 2, 2>(a, s) : launch_grouped<E, 128, 128, 2, 2>(a, s);
}

}  // namespace

extern "C" {

// Rows of an m tile: what the routing's tile list has to be made for.
int nf_grouped_tile_rows(int dtype, int rows, int groups) {
  if (dtype == NF_F32) return kF32Tile;
  return (long long)rows <= 96ll * std::max(groups, 1) ? 64 : 128;
}

int nf_gemm_grouped(const nf_grouped_gemm_args* args, nf_stream_t stream) {
  const char* who = "nf_gemm_grouped";
  NF_REQUIRE(args, "%s: null pointer", who);
  const nf_grouped_gemm_args& a = *args;
  NF_REQUIRE(a.dtype == NF_F32 || a.dtype == NF_BF16, "%s: unknown dtype %d", who, a.dtype);
  NF_REQUIRE(a.act == NF_ACT_NONE || a.act == NF_ACT_GELU || a.act == NF_ACT_SQUARED_RELU || a.act == NF_ACT_GATED, "%s: unknown activation %d", who, a.act);
  NF_REQUIRE(a.groups > 0 && a.M >= 0 && a.N > 0 && a.K > 0 && a.N % 8 == 0 && a.K % 8 == 0 && a.lda >= a.K && a.ldd >= (a.act == NF_ACT_GATED ? a.N / 2 : a.N) && a.lda % 8 == 0 &&
                 a.ldd % 8 == 0 && a.a_group % 8 == 0 && a.d_group % 8 == 0,
             "%s: bad shape: %d groups, M=%d N=%d K=%d, strides %d %d", who, a.groups, a.M, a.N, a.K, a.lda, a.ldd);
  const bool routed = a.routing.n_tiles != nullptr;
  NF_REQUIRE(!routed || (a.routing.tile_group && a.routing.tile_row && a.routing.offsets && a.max_rows >= 0 && (!a.gather || a.routing.row_of)),
             "%s: incomplete routing", who);
  NF_REQUIRE(!a.weigh || (routed && a.routing.row_weight), "%s: no weights of the sorted rows", who);
  if (a.M == 0 || (routed && a.max_rows == 0)) return NF_OK;
  NF_REQUIRE(a.a && a.b && a.d, "%s: null pointer", who);
  NF_REQUIRE(((uintptr_t)a.a | (uintptr_t)a.b | (uintptr_t)a.d) % 16 == 0, "%s: operands must be 16-byte aligned", who);
  const int a_rows = routed && !a.gather ? a.max_rows : a.M;
  NF_REQUIRE(((size_t)a_rows + 256) * ((size_t)a.lda + 512) * 2 < 0xFFFFFF00ull && ((size_t)a.N + 256) * ((size_t)a.K + 512) * 2 < 0xFFFFFF00ull,
             "%s: an operand exceeds the 4 GiB buffer-addressing limit", who);
  const int tile_rows = nf_grouped_tile_rows(a.dtype, routed ? a.max_rows : a.M * a.groups, a.groups);
  NF_REQUIRE(!routed || a.routing.tile_rows == tile_rows, "%s: the tile list is for tiles of %d rows, not %d", who, a.routing.tile_rows, tile_rows);
  hipStream_t s = (hipStream_t)stream;
  if (a.dtype == NF_F32) {
    const int tiles_n = (a.N + kF32Tile - 1) / kF32Tile;
    auto kern = a.act == NF_ACT_GELU           ? gemm_grouped_f32_kernel<NF_ACT_GELU>
                : a.act == NF_ACT_SQUARED_RELU ? gemm_grouped_f32_kernel<NF_ACT_SQUARED_RELU>
                : a.act == NF_ACT_GATED        ? gemm_grouped_f32_kernel<NF_ACT_GATED>
                                               : gemm_grouped_f32_kernel<NF_ACT_NONE>;
    kern<<<grid_of(a, kF32Tile, tiles_n), 256, 0, s>>>(a, tiles_n);
    return check_launch(who);
  }
  if (a.act == NF_ACT_SQUARED_RELU) return dispatch_grouped<BF16SquaredRelu>(a, tile_rows, s);
  if (a.act == NF_ACT_GATED) return dispatch_grouped<BF16Gated>(a, tile_rows, s);
  return a.act == NF_ACT_GELU ? dispatch_grouped<BF16Gelu>(a, tile_rows, s) : dispatch_grouped<BF16>(a, tile_rows, s);
}

}  // extern "C"
