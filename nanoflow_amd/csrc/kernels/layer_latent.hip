// Latent attention of the layer-stack pipeline: the cache holds one latent row and one rotated key part per
// position for all heads, queries come already multiplied into the latent space, and the values are the latents
// themselves -- so attention is one set of keys and values under (tokens x heads) query columns.
//
// bf16 (latent_mfma_kernel, v_mfma_f32_16x16x32_bf16): S^T = K . Q^T, then O^T = C^T . P^T with C the
// latent part of the same rows.
//   * A workgroup's columns -- consecutive (token, head) pairs of a request, `cbs` blocks of 16 -- share 32-key tiles
//     that go straight into LDS (buffer_load ... lds), a ring of four.  A tile lies there in planes of 64 elements:
//     32 rows of 128 bytes, 16-byte chunk c of row r at position c ^ f(r) with f = the bits (r>>1 & 3, r>>3 & 1): the 16
//     rows of a key fragment fall on 16 different 16-byte slots, and the rows of two groups' transposing reads
//     (ds_read_b64_tr_b16) on eight different 32-byte ones.
//   * 2 x cbs wavefronts.  For the scores each takes 16 of the keys and one block of columns, for the product with the values
//     a part of the value columns and all blocks; maxima and weights pass between the two through LDS.  So nothing is
//     computed or read twice but by that exchange, and 512 value columns of four blocks fit the registers.
//   * The scores of a tile and the value product of the tile before it stand between the same two barriers.
//   * Softmax weights keep 32 bits: P is multiplied as two bf16 terms, P = hi + lo.
//   * `splits` > 1: workgroups share a request's tiles and leave (m, l, O) for latent_merge_kernel.
// fp32, and sizes beyond the tiles (latent_rows_kernel): one wavefront per (row, head), every product in 32-bit.
#include <algorithm>
#include <cmath>

#include "layer_common.h"

namespace nf {

constexpr int kLatentPage = 16, kTileKeys = 32, kRing = 4, kMaxSplits = 16;
constexpr int kMaxRank = 2048, kMaxRowLd = 2304;
constexpr float kLog2e = 1.44269504088896340736f;

template <class T>
__device__ __forceinline__ float turned(const T* src, int d, const nf_rotation& rot, int pos) {
  const float y = Act<T>::load(src + d);
  const int half = rot.dims / 2;
  if (d >= 2 * half) return y;
  const int f = rot.interleaved ? d >> 1 : (d < half ? d : d - half);
  const bool first = rot.interleaved ? !(d & 1) : d < half;
  const float other = Act<T>::load(src + (rot.interleaved ? d ^ 1 : (first ? d + half : d - half)));
  const float cs = rot.table[((size_t)pos * half + f) * 2], sn = rot.table[((size_t)pos * half + f) * 2 + 1];
  return first ? y * cs - other * sn : y * cs + other * sn;
}

// One workgroup per row.
template <class T>
__global__ __launch_bounds__(256) void latent_append_kernel(nf_latent_layout lay, const T* __restrict__ proj, int ld, int q_col, int kv_col,
                                                            const float* __restrict__ norm, float eps, nf_rotation rot, T* __restrict__ q,
                                                            T* __restrict__ kv_data, const int32_t* __restrict__ kv_indptr,
                                                            const int32_t* __restrict__ kv_indices,
                                                            const int32_t* __restrict__ rev_input_indptr,
                                                            const int32_t* __restrict__ positions, int q_rows) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, tid = threadIdx.x, pos = positions[t];
  const int page = kv_indices[kv_indptr[rev_input_indptr[t]] + pos / kLatentPage];
  const T* src = proj + (size_t)t * ld;
  T* dst = kv_data + ((size_t)page * kLatentPage + pos % kLatentPage) * lay.row_ld;
  float c[kMaxRank / 256], sq = 0.f;
#pragma unroll
  for (int i = 0; i < kMaxRank / 256; ++i) {
    const int e = i * 256 + tid;
    c[i] = e < lay.kv_rank ? Act<T>::load(src + kv_col + e) : 0.f;
    sq += c[i] * c[i];
  }
  const float inv = 1.f / sqrtf(block_sum(sq, scratch) / (float)lay.kv_rank + eps);
#pragma unroll
  for (int i = 0; i < kMaxRank / 256; ++i) {
    const int e = i * 256 + tid;
    if (e < lay.rank_pad) Act<T>::store(dst + e, e < lay.kv_rank ? c[i] * inv * norm[e] : 0.f);
  }
  const int tail = lay.row_ld - lay.rank_pad;  // rotated part and padding
  if (rot.interleaved && (lay.rot_dim | rot.dims | ld | q_col | kv_col | lay.kv_rank) % 4 == 0) {  // four elements at a time
    const float* tab = rot.table + (size_t)pos * rot.dims;
    const int quads = tail / 4, all = t < q_rows ? (lay.heads + 1) * quads : quads;
    for (int e = tid; e < all; e += 256) {
      const int h = e / quads - 1, d = e % quads * 4;  // head -1 is the key's part
      const bool key = h < 0;
      float4_t v{0.f, 0.f, 0.f, 0.f};
      if (d < lay.rot_dim) v = Act<T>::load4(src + (key ? kv_col + lay.kv_rank : q_col + h * lay.rot_dim) + d);
      if (d < rot.dims) {
        const float4_t cs = *reinterpret_cast<const float4_t*>(tab + d);
        v = float4_t{v[0] * cs[0] - v[1] * cs[1], v[1] * cs[0] + v[0] * cs[1], v[2] * cs[2] - v[3] * cs[3], v[3] * cs[2] + v[2] * cs[3]};
      }
      Act<T>::store4((key ? dst : q + ((size_t)t * lay.heads + h) * lay.row_ld) + lay.rank_pad + d, v);
    }
    return;
  }
  for (int e = tid; e < tail; e += 256)
    Act<T>::store(dst + lay.rank_pad + e, e < lay.rot_dim ? turned(src + kv_col + lay.kv_rank, e, rot, pos) : 0.f);
  if (t >= q_rows) return;
  for (int e = tid; e < lay.heads * tail; e += 256) {
    const int h = e / tail, d = e % tail;
    Act<T>::store(q + ((size_t)t * lay.heads + h) * lay.row_ld + lay.rank_pad + d,
                  d < lay.rot_dim ? turned(src + q_col + h * lay.rot_dim, d, rot, pos) : 0.f);
  }
}

// ---------------------------------------------------------------- keys and values written out
// One workgroup per page of the requests.
template <class T>
__global__ __launch_bounds__(256) void latent_gather_kernel(nf_latent_expand_args a) {
  const int R = a.layout.rank_pad, first = a.kv_indptr[a.req_begin], at = first + blockIdx.x;
  const bool live = at < a.kv_indptr[a.req_end];
  const T* src = (const T*)a.kv_data + (size_t)(live ? a.kv_indices[at] : 0) * kLatentPage * a.layout.row_ld;
  T* dst = (T*)a.rows + (size_t)blockIdx.x * kLatentPage * R;
  if (live && threadIdx.x == 0) a.page_ids[at] = blockIdx.x;
  for (int e = threadIdx.x; e < kLatentPage * R / 4; e += 256) {
    const int r = e / (R / 4), c = e % (R / 4) * 4;
    Act<T>::store4(dst + (size_t)r * R + c, live ? Act<T>::load4(src + (size_t)r * a.layout.row_ld + c) : float4_t{0.f, 0.f, 0.f, 0.f});
  }
}

// One workgroup per (head, page): rows are read in four-element groups; V is turned through LDS.
template <class T>
__global__ __launch_bounds__(256) void latent_pack_kernel(nf_latent_expand_args a) {
  __shared__ float turn[kLatentPage * 260];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x, at = a.kv_indptr[a.req_begin] + b;
  if (at >= a.kv_indptr[a.req_end]) return;
  const nf_kv_layout kv = a.kv;
  const int tail = a.layout.row_ld - a.layout.rank_pad;
  const T* cached = (const T*)a.kv_data + (size_t)a.kv_indices[at] * kLatentPage * a.layout.row_ld + a.layout.rank_pad;
  const T* prod = (const T*)a.products + (size_t)b * kLatentPage * a.ld;
  T* page = (T*)a.pages + (size_t)b * kv.heads * kLatentPage * (kv.k_pad + kv.v_pad);
  for (int e = tid; e < kLatentPage * kv.v_pad / 4; e += 256) {
    const int r = e / (kv.v_pad / 4), c = e % (kv.v_pad / 4) * 4;
    float4_t v{0.f, 0.f, 0.f, 0.f};
    if (c < kv.vdim) v = Act<T>::load4(prod + (size_t)r * a.ld + a.v_col + h * kv.vdim + c);
#pragma unroll
    for (int x = 0; x < 4; ++x) turn[r * 260 + c + x] = v[x];
  }
  T* k_page = page + (size_t)h * kLatentPage * kv.k_pad;
  for (int e = tid; e < kLatentPage * kv.k_pad / 4; e += 256) {
    const int r = e / (kv.k_pad / 4), c = e % (kv.k_pad / 4) * 4, d = c - a.dim_pad;
    float4_t v{0.f, 0.f, 0.f, 0.f};
    if (d < 0) v = Act<T>::load4(prod + (size_t)r * a.ld + a.k_col + h * a.dim_pad + c);
    else if (d < tail) v = Act<T>::load4(cached + (size_t)r * a.layout.row_ld + d);  // zero behind the rotated part
    Act<T>::store4(k_page + (size_t)r * kv.k_pad + c, v);
  }
  __syncthreads();
  T* v_page = page + (size_t)kv.heads * kLatentPage * kv.k_pad + (size_t)h * kv.v_pad * kLatentPage;
  for (int e = tid; e < kv.v_pad * 4; e += 256) {
    const int c = e >> 2, r = (e & 3) * 4;
    Act<T>::store4(v_page + (size_t)c * kLatentPage + r,
                   float4_t{turn[r * 260 + c], turn[(r + 1) * 260 + c], turn[(r + 2) * 260 + c], turn[(r + 3) * 260 + c]});
  }
}

// One workgroup per row.
template <class T>
__global__ __launch_bounds__(256) void latent_queries_kernel(nf_kv_layout kv, int dim_pad, const T* __restrict__ proj, int ld, int q_col, int rot_dim,
                                                             nf_rotation rot, const int32_t* __restrict__ positions, T* __restrict__ q,
                                                             int row_begin) {
  const int t = row_begin + blockIdx.x, pos = positions[t];
  const T* src = proj + (size_t)t * ld;
  T* dst = q + (size_t)t * kv.heads * kv.k_pad;
  const bool four = rot.interleaved && (rot_dim | rot.dims | ld | q_col) % 4 == 0;
  const float* tab = rot.table + (size_t)pos * rot.dims;
  for (int e = threadIdx.x; e < kv.heads * kv.k_pad / 4; e += 256) {
    const int h = e / (kv.k_pad / 4), c = e % (kv.k_pad / 4) * 4, d = c - dim_pad;
    float4_t v{0.f, 0.f, 0.f, 0.f};
    if (d < 0) {
      v = Act<T>::load4(src + h * dim_pad + c);
    } else if (four && d < rot_dim) {
      v = Act<T>::load4(src + q_col + h * rot_dim + d);
      if (d < rot.dims) {
        const float4_t cs = *reinterpret_cast<const float4_t*>(tab + d);
        v = float4_t{v[0] * cs[0] - v[1] * cs[1], v[1] * cs[0] + v[0] * cs[1], v[2] * cs[2] - v[3] * cs[3], v[3] * cs[2] + v[2] * cs[3]};
      }
    } else {
#pragma unroll
      for (int x = 0; x < 4; ++x)
        if (d + x < rot_dim) v[x] = turned(src + q_col + h * rot_dim, d + x, rot, pos);
    }
    Act<T>::store4(dst + h * kv.k_pad + c, v);
  }
}

// The first position that one at p sees.
__device__ __forceinline__ int first_seen(int p, int window) { return window > 0 && p >= window ? p - window + 1 : 0; }

// ---------------------------------------------------------------- fp32, any size
template <class T, int NE>  // NE x 64 latent columns at most
__global__ __launch_bounds__(64) void latent_rows_kernel(nf_latent_attention_args a) {
  __shared__ __attribute__((aligned(16))) float sq[kMaxRowLd];
  __shared__ float sp[64];
  const nf_latent_layout lay = a.layout;
  const int lane = threadIdx.x, t = a.row_begin + blockIdx.x, h = blockIdx.y;
  const int req = a.rev_input_indptr[t], p = a.positions[t];
  const T* q = (const T*)a.q + ((size_t)t * lay.heads + h) * lay.row_ld;
  for (int c = lane; c < lay.row_ld; c += 64) sq[c] = Act<T>::load(q + c);
  __syncthreads();
  const int32_t* pages = a.kv_indices + a.kv_indptr[req];
  auto row_of = [&](int j) { return (const T*)a.kv_data + ((size_t)pages[j / kLatentPage] * kLatentPage + j % kLatentPage) * lay.row_ld; };
  float m = -1e30f, l = 0.f, o[NE] = {};
  for (int base = first_seen(p, a.window) / 64 * 64; base <= p; base += 64) {
    const int j = base + lane;
    const bool see = j <= p && j >= first_seen(p, a.window);
    float s = -INFINITY;
    if (see) {
      const T* k = row_of(j);
      float dot = 0.f;
      for (int c = 0; c < lay.row_ld; c += 4) {
        const float4_t kk = Act<T>::load4(k + c), qq = *reinterpret_cast<const float4_t*>(sq + c);
        dot += kk[0] * qq[0] + kk[1] * qq[1] + kk[2] * qq[2] + kk[3] * qq[3];
      }
      s = dot * a.scale;
    }
    float mx = s;
#pragma unroll
    for (int d = 32; d > 0; d >>= 1) mx = fmaxf(mx, __shfl_xor(mx, d, 64));
    const float m_new = fmaxf(m, mx), alpha = expf(m - m_new), w = see ? expf(s - m_new) : 0.f;
    m = m_new;
    l = l * alpha + w;
    __syncthreads();
    sp[lane] = w;
    __syncthreads();
#pragma unroll
    for (int e = 0; e < NE; ++e) o[e] *= alpha;
    const int n = min(64, p - base + 1);
    for (int r = 0; r < n; ++r) {
      const T* v = row_of(base + r);
      const float wt = sp[r];
#pragma unroll
      for (int e = 0; e < NE; ++e)
        if (e * 64 + lane < lay.rank_pad) o[e] += wt * Act<T>::load(v + e * 64 + lane);
    }
  }
  const float inv = 1.f / wave_sum(l);
  T* out = (T*)a.out + ((size_t)t * lay.heads + h) * lay.rank_pad;
#pragma unroll
  for (int e = 0; e < NE; ++e)
    if (e * 64 + lane < lay.rank_pad) Act<T>::store(out + e * 64 + lane, o[e] * inv);
}

// ---------------------------------------------------------------- bf16
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
union L8 {
  u32x4 u;
  bf16x8_t b;
  uint32_t w[4];
};

struct LatentLaunch {
  int splits, tiles_per_request;  // tiles_per_request: decoding; 0 in prompts
  float* part_o;                  // [row][head][split][rank_pad]
  float* part_ml;                 // [row][head][split][2]
};

template <int CBS>
struct LatentShared {
  uint32_t p[CBS][2][64][4];  // weights, high and low terms, as a lane of the value product takes them
  float mx[2][CBS][16], l[2][CBS][16];
};

// KD: 32-wide pieces of row_ld, VD: 16-wide value tiles; upper bounds, or (kExact) the sizes themselves.
template <int KD, int VD, int CBS, bool kExact>
__global__ __launch_bounds__(CBS * 128) void latent_mfma_kernel(nf_latent_attention_args a, LatentLaunch p) {
  constexpr int kWaves = 2 * CBS, VW = (VD + kWaves - 1) / kWaves;  // value tiles of a wavefront
  extern __shared__ __attribute__((aligned(1024))) uint8_t tile_lds[];
  const uint32_t lds0 = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) uint8_t*)tile_lds;
  const nf_latent_layout lay = a.layout;
  const uint32_t slot_bytes = (uint32_t)kTileKeys * lay.row_ld * 2;
  LatentShared<CBS>& sh = *reinterpret_cast<LatentShared<CBS>*>(tile_lds + kRing * slot_bytes);
  const int H = lay.heads, lane = threadIdx.x & 63, l16 = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int cb = wave % CBS, kt = wave / CBS, v0 = wave * VW;  // scores: column block, 16-key half; values: first tile
  constexpr int columns = CBS * 16;

  const bool decode = p.tiles_per_request > 0;
  int req = -1, tile = blockIdx.x;
  if (decode) {
    req = a.req_begin + tile / p.tiles_per_request;  // one row each
    tile %= p.tiles_per_request;
  } else {
    for (int r = a.req_begin; r < a.req_begin + a.req_num; ++r) {
      const int n = ((a.input_indptr[r + 1] - a.input_indptr[r]) * H + columns - 1) / columns;
      if (tile < n) {
        req = r;
        tile = n - 1 - tile;  // the tiles that see most keys start first
        break;
      }
      tile -= n;
    }
    if (req < 0) return;
  }
  const int row0 = decode ? a.row_begin + req - a.req_begin : a.input_indptr[req], len = decode ? 1 : a.input_indptr[req + 1] - row0;
  const int col0 = tile * columns, total = len * H;
  const int pos0 = a.positions[row0];
  const int p_low = pos0 + col0 / H, p_high = pos0 + min(col0 + columns - 1, total - 1) / H;

  const int kd = kExact ? KD : lay.row_ld / 32, vd = kExact ? VD : (lay.rank_pad + 15) / 16, planes = kExact ? KD / 2 : lay.row_ld / 64;
  const int first_tile = first_seen(p_low, a.window) / kTileKeys;  // tiles before it are out of every column's window
  const int end_tile = p_high / kTileKeys + 1, per = (end_tile - first_tile + p.splits - 1) / p.splits;
  const int t0 = first_tile + blockIdx.y * per, t1 = min(end_tile, t0 + per);
  const int32_t* pages = a.kv_indices + a.kv_indptr[req];
  const int last_page = p_high / kLatentPage;
  const size_t page_bytes = (size_t)kLatentPage * lay.row_ld * 2;

  // Page ids of 32 tiles at a time, two per tile, one per lane: a load of its own in every tile would wait for all the tiles
  // in flight.
  int ids = 0;
  auto load_ids = [&](int t) {
    ids = pages[min(t * (kTileKeys / kLatentPage) + lane, last_page)];
    __builtin_amdgcn_s_waitcnt(0x0F70);
  };
  // One load instruction fills 8 keys of one plane.  Two wavefronts: every second group of 8 keys each; four: a group each; eight:
  // a group and every second plane of it.
  const int r8 = lane >> 3;
  constexpr int kPlaneStep = kWaves == 8 ? 2 : 1;
  auto load_tile = [&](int t) {
    if ((t - t0) % 32 == 0) load_ids(t);
#pragma unroll
    for (int rg = wave & 3; rg < 4; rg += kWaves < 4 ? kWaves : 4) {
      const int page = __builtin_amdgcn_readlane(ids, (t - t0) % 32 * 2 + rg / 2);
      const rsrc_t rsrc = make_rsrc((const uint8_t*)a.kv_data + (size_t)page * page_bytes, page_bytes);
      const int chunk = (lane & 7) ^ (((r8 >> 1) << 1) | (rg & 1)), pl0 = kWaves == 8 ? wave >> 2 : 0;
      uint32_t off = (uint32_t)((rg & 1) * 8 + r8) * (uint32_t)lay.row_ld * 2u + (uint32_t)chunk * 16u + (uint32_t)pl0 * 128u;
      uint32_t at = __builtin_amdgcn_readfirstlane(lds0 + (uint32_t)((t - t0) % kRing) * slot_bytes + (uint32_t)pl0 * (kTileKeys * 128) + (uint32_t)rg * 1024u);
      for (int pl = pl0; pl < planes; pl += kPlaneStep) {
        // up to two blocks, decoding only: every row is read once, the hint keeps it from displacing what the caches hold
        if constexpr (CBS <= 2) load16_to_lds_nt(rsrc, off, at);
        else load16_to_lds(rsrc, off, at);
        off += kPlaneStep * 128;
        at += kPlaneStep * kTileKeys * 128;
      }
    }
  };
  // Waits until this wavefront's loads of tile t have landed; the next tile's may still be in flight (their number is known
  // where the size is; a wavefront that takes more planes than another waits longer).
  constexpr int kLoads = kWaves == 2 ? KD : kWaves == 4 ? KD / 2 : KD / 4;
  auto wait_tile = [&](int t) {
    if (kExact && t + 1 < t1) __builtin_amdgcn_s_waitcnt(0x0F70 | (kLoads & 15) | ((kLoads >> 4) << 14));
    else __builtin_amdgcn_s_waitcnt(0x0F70);
  };

  float4_t o[CBS][VW];
  float m[CBS], l = 0.f;  // l: of this wavefront's keys
#pragma unroll
  for (int c = 0; c < CBS; ++c) {
    m[c] = -1e30f;
#pragma unroll
    for (int i = 0; i < VW; ++i) o[c][i] = float4_t{0.f, 0.f, 0.f, 0.f};
  }
  const float scale2 = a.scale * kLog2e;
  // LDS offsets of this lane's pieces: key row 16 kt + l16, chunk (j & 1) * 4 + g of plane j / 2; value rows 4g + l16 / 4
  const uint32_t kf_swz = (uint32_t)((((l16 >> 1) & 3) << 1) | (l16 >> 3));
  const uint32_t k_row = (uint32_t)(kt * 16 + l16) * 128u;
  const uint32_t kx[2] = {k_row + (((uint32_t)g ^ kf_swz) << 4), k_row + (((uint32_t)(4 + g) ^ kf_swz) << 4)};
  const int vrow = 4 * g + (l16 >> 2), vj = (vrow >> 1) & 7;
  const uint32_t v_swz = (uint32_t)(((vj & 3) << 1) | (vj >> 2));
  uint32_t vx[4];
#pragma unroll
  for (int u = 0; u < 4; ++u)
    vx[u] = (uint32_t)vrow * 128u + (((uint32_t)(2 * u + ((l16 & 3) >> 1)) ^ v_swz) << 4) + (uint32_t)(l16 & 1) * 8u;

#pragma unroll 1
  for (int t = t0; t < min(t0 + 2, t1); ++t) load_tile(t);
  int pos;
  L8 qf[KD];
  {
    const int col = col0 + cb * 16 + l16;
    const bool live = col < total;  // the others see no key; what they multiply does not matter
    pos = live ? pos0 + col / H : -1;
    const bf16_t* q = (const bf16_t*)a.q + ((size_t)(row0 + (live ? col / H : 0)) * H + (live ? col % H : 0)) * lay.row_ld + g * 8;
#pragma unroll
    for (int j = 0; j < KD; ++j) qf[j].u = kExact || j < kd ? *reinterpret_cast<const u32x4*>(q + j * 32) : u32x4{0, 0, 0, 0};
  }
  // Everything has landed once, here: a wait for the queries inside the loop would be one for the tiles in flight.
  __builtin_amdgcn_s_waitcnt(0x0F70);

  // This wavefront's 16 keys of a tile against its block: two sums, so that an MFMA does not wait for the one before it.
  auto scores = [&](const uint8_t* slot) {
    float4_t s[2] = {float4_t{0.f, 0.f, 0.f, 0.f}, float4_t{0.f, 0.f, 0.f, 0.f}};
    constexpr int kStep = 6, kSteps = (KD + kStep - 1) / kStep;  // pieces requested together
    L8 kf[2][kStep];
    auto read = [&](int c) {
#pragma unroll
      for (int x = 0; x < kStep; ++x) {
        const int j = c * kStep + x;
        if (j < KD && (kExact || j < kd)) kf[c & 1][x].u = *reinterpret_cast<const u32x4*>(slot + (j >> 1) * (kTileKeys * 128) + kx[j & 1]);
      }
    };
    read(0);
#pragma unroll
    for (int c = 0; c < kSteps; ++c) {
      if (c + 1 < kSteps) read(c + 1);
#pragma unroll
      for (int x = 0; x < kStep; ++x) {
        const int j = c * kStep + x;
        if (j < KD && (kExact || j < kd)) s[x & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[c & 1][x].b, qf[j].b, s[x & 1], 0, 0, 0);
      }
    }
    return s[0] + s[1];
  };
  // All columns' weights of a tile against this wavefront's value tiles.
  auto values = [&](const uint8_t* slot) {
    L8 w[CBS][2];
#pragma unroll
    for (int c = 0; c < CBS; ++c)
#pragma unroll
      for (int x = 0; x < 2; ++x) w[c][x].u = *reinterpret_cast<const u32x4*>(sh.p[c][x][lane]);
#pragma unroll
    for (int i = 0; i < VW; ++i) {
      const int vt = v0 + i;
      if (!kExact && vt >= vd) continue;
      const uint8_t* v = slot + (vt >> 2) * (kTileKeys * 128) + (VW % 4 == 0 ? vx[i & 3] : vx[vt & 3]);
      const short4_t a0 = lds_read_tr16(v), a1 = lds_read_tr16(v + 2048);
      typedef short short8_t __attribute__((ext_vector_type(8)));
      const bf16x8_t vf = __builtin_bit_cast(bf16x8_t, (short8_t)__builtin_shufflevector(a0, a1, 0, 1, 2, 3, 4, 5, 6, 7));
#pragma unroll
      for (int x = 0; x < 2; ++x)
#pragma unroll
        for (int c = 0; c < CBS; ++c) o[c][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, w[c][x].b, o[c][i], 0, 0, 0);
    }
  };
  auto slot_of = [&](int t) { return (const uint8_t*)tile_lds + (size_t)((t - t0) % kRing) * slot_bytes; };

#pragma unroll 1
  for (int t = t0; t < t1; ++t) {
    wait_tile(t);
    __syncthreads();  // the tile has landed, the weights of the one before it are written, and the one before that is done with
    if (t + 2 < t1) load_tile(t + 2);
    if (t > t0) values(slot_of(t - 1));
    float4_t s = scores(slot_of(t));
    const int base = t * kTileKeys + kt * 16 + 4 * g;
    if (t * kTileKeys + 31 > p_low)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (base + r > pos) s[r] = -INFINITY;
    if (a.window > 0 && t * kTileKeys <= p_high - a.window)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (base + r <= pos - a.window) s[r] = -INFINITY;
    float mx = fmaxf(fmaxf(s[0], s[1]), fmaxf(s[2], s[3]));
    mx = max_over_lane_groups(mx > -1e30f ? mx * scale2 : -1e30f);
    if (g == 0) sh.mx[kt][cb][l16] = mx;
    __syncthreads();  // everyone's maxima are there, and the weights of the tile before have been read
    float my_m = 0.f;
#pragma unroll
    for (int c = 0; c < CBS; ++c) {
      // The sums are brought to a new maximum only when it has grown by 2^8: until then weights are up to 256, which
      // costs nothing in fp32.  Every wavefront decides the same from the same maxima.
      const float both = fmaxf(sh.mx[0][c][l16], sh.mx[1][c][l16]);
      if (__any(both > m[c] + 8.f)) {
        const float m_new = fmaxf(m[c], both), alpha = __builtin_amdgcn_exp2f(m[c] - m_new);
        m[c] = m_new;
        if (c == cb) l *= alpha;
#pragma unroll
        for (int i = 0; i < VW; ++i) o[c][i] *= alpha;
      }
      if (c == cb) my_m = m[c];
    }
    uint32_t hi[2], lo[2];
#pragma unroll
    for (int r = 0; r < 4; r += 2) {
      const float w0 = __builtin_amdgcn_exp2f(fmaf(s[r], scale2, -my_m)), w1 = __builtin_amdgcn_exp2f(fmaf(s[r + 1], scale2, -my_m));
      l += w0 + w1;
      hi[r / 2] = f32_to_bf16_pair(w0, w1);
      lo[r / 2] = f32_to_bf16_pair(w0 - __uint_as_float(hi[r / 2] << 16), w1 - __uint_as_float(hi[r / 2] & 0xffff0000u));
    }
    *reinterpret_cast<u32x2*>(&sh.p[cb][0][lane][kt * 2]) = u32x2{hi[0], hi[1]};
    *reinterpret_cast<u32x2*>(&sh.p[cb][1][lane][kt * 2]) = u32x2{lo[0], lo[1]};
  }
  l = sum_over_lane_groups(l);
  if (g == 0) sh.l[kt][cb][l16] = l;
  __syncthreads();
  if (t0 < t1) values(slot_of(t1 - 1));

#pragma unroll
  for (int c = 0; c < CBS; ++c) {
    const int col = col0 + c * 16 + l16;
    if (col >= total) continue;
    const int row = row0 + col / H, head = col % H;
    const float den = sh.l[0][c][l16] + sh.l[1][c][l16];
    if (p.splits > 1) {
      const size_t at = ((size_t)(row - a.row_begin) * H + head) * p.splits + blockIdx.y;
      if (g == 0 && wave == 0) {
        p.part_ml[at * 2] = m[c];
        p.part_ml[at * 2 + 1] = den;
      }
      float* dst = p.part_o + at * lay.rank_pad;
#pragma unroll
      for (int i = 0; i < VW; ++i)
        if ((v0 + i) * 16 + g * 4 < lay.rank_pad) *reinterpret_cast<float4_t*>(dst + (v0 + i) * 16 + g * 4) = o[c][i];
    } else {
      const float inv = 1.f / den;
      bf16_t* dst = (bf16_t*)a.out + ((size_t)row * H + head) * lay.rank_pad;
#pragma unroll
      for (int i = 0; i < VW; ++i)
        if ((v0 + i) * 16 + g * 4 < lay.rank_pad) Act<bf16_t>::store4(dst + (v0 + i) * 16 + g * 4, o[c][i] * inv);
    }
  }
}

// One wavefront per (row, head): the splits' sums brought to a common maximum.
__global__ __launch_bounds__(256) void latent_merge_kernel(nf_latent_attention_args a, LatentLaunch p, int pairs) {
  const int lane = threadIdx.x & 63, pair = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (pair >= pairs) return;
  const int R = a.layout.rank_pad, at = lane < p.splits ? lane : 0;
  const float* ml = p.part_ml + (size_t)pair * p.splits * 2;
  const float m = lane < p.splits ? ml[2 * at] : -1e30f, l = lane < p.splits ? ml[2 * at + 1] : 0.f;
  float mm = m;
#pragma unroll
  for (int d = 32; d > 0; d >>= 1) mm = fmaxf(mm, __shfl_xor(mm, d, 64));
  const float den = wave_sum(l * __builtin_amdgcn_exp2f(m - mm));
  const float f = l > 0.f ? __builtin_amdgcn_exp2f(m - mm) / den : 0.f;  // 0: a share whose keys are all unseen
  bf16_t* dst = (bf16_t*)a.out + ((size_t)a.row_begin * a.layout.heads + pair) * R;
  const float* o = p.part_o + (size_t)pair * p.splits * R;
  constexpr int kAhead = 4;
  for (int c0 = 0; c0 < R; c0 += 256) {  // every lane stays: the factors come from other lanes
    const int c = c0 + lane * 4, cc = c < R ? c : 0;
    float4_t v{0.f, 0.f, 0.f, 0.f};
    for (int s0 = 0; s0 < p.splits; s0 += kAhead) {
      float4_t x[kAhead];
#pragma unroll
      for (int s = 0; s < kAhead; ++s) x[s] = *reinterpret_cast<const float4_t*>(o + (size_t)min(s0 + s, p.splits - 1) * R + cc);
#pragma unroll
      for (int s = 0; s < kAhead; ++s) {
        const float fs = __shfl(f, min(s0 + s, 63), 64);  // 0 past the last share
        if (fs > 0.f) v += x[s] * fs;
      }
    }
    if (c < R) Act<bf16_t>::store4(dst + c, v);
  }
}

template <int KD, int VD, int CBS, bool kExact>
static int launch_blocks(const nf_latent_attention_args& a, hipStream_t s) {
  const int H = a.layout.heads;
  LatentLaunch p{};
  if (a.decode) p.tiles_per_request = (H + CBS * 16 - 1) / (CBS * 16);
  const long long tiles = a.decode ? (long long)a.req_num * p.tiles_per_request : (long long)a.max_rows * H / (CBS * 16) + a.req_num;
  const size_t lds = (size_t)kRing * kTileKeys * a.layout.row_ld * 2 + sizeof(LatentShared<CBS>);
  // as many workgroups as the CUs hold at a time, one or two each
  const size_t per_split = (size_t)a.max_rows * H * (a.layout.rank_pad + 2) * sizeof(float);
  p.splits = (int)std::min<long long>(kMaxSplits, std::max<long long>((lds > 80 * 1024 ? 256 : 512) / tiles, 1));
  p.splits = std::max(1, (int)std::min<size_t>((size_t)p.splits, a.workspace ? a.workspace_bytes / per_split : 0));
  if (p.splits > 1) {
    p.part_o = (float*)a.workspace;
    p.part_ml = p.part_o + (size_t)a.max_rows * H * p.splits * a.layout.rank_pad;
  }
  auto kern = latent_mfma_kernel<KD, VD, CBS, kExact>;
  static size_t reserved = 0;  // benign race: the call is idempotent
  if (lds > reserved) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) {
      set_error("nf_latent_attention: cannot reserve %zu bytes of LDS: %s", lds, hipGetErrorString(e));
      return NF_ERR_RUNTIME;
    }
    reserved = lds;
  }
  kern<<<dim3((unsigned)tiles, (unsigned)p.splits), CBS * 128, lds, s>>>(a, p);
  int rc = check_launch("nf_latent_attention");
  if (rc || p.splits == 1) return rc;
  const int pairs = a.max_rows * H;
  latent_merge_kernel<<<(pairs + 3) / 4, 256, 0, s>>>(a, p, pairs);
  return check_launch("nf_latent_attention (merge)");
}

template <int KD, int VD, bool kExact>
static int launch_latent(const nf_latent_attention_args& a, hipStream_t s) {
  if (a.decode && a.layout.heads <= 16) return launch_blocks<KD, VD, 1, kExact>(a, s);
  if (a.decode && a.layout.heads <= 32) return launch_blocks<KD, VD, 2, kExact>(a, s);
  return launch_blocks<KD, VD, 4, kExact>(a, s);
}

}  // namespace nf

using namespace nf;

static int check_latent(const char* who, const nf_latent_layout& l) {
  NF_REQUIRE(l.dtype == NF_F32 || l.dtype == NF_BF16, "%s: unknown dtype %d", who, l.dtype);
  NF_REQUIRE(l.heads > 0 && l.heads <= 65535 && l.kv_rank > 0 && l.kv_rank <= kMaxRank && l.rot_dim >= 0 && l.rot_dim <= 256 &&
                 l.page == kLatentPage && l.rank_pad == (l.kv_rank + 7) / 8 * 8 && l.row_ld == (l.rank_pad + l.rot_dim + 63) / 64 * 64,
             "%s: %d heads, latent size %d (pad %d), %d rotated (rows of %d), page %d: pages of 16, latents up to %d", who, l.heads, l.kv_rank,
             l.rank_pad, l.rot_dim, l.row_ld, l.page, kMaxRank);
  return NF_OK;
}

extern "C" {

int nf_latent_layout_of(int dtype, int heads, int kv_rank, int rot_dim, int page, nf_latent_layout* out) {
  NF_REQUIRE(out, "nf_latent_layout_of: null pointer");
  *out = nf_latent_layout{dtype, heads, kv_rank, (kv_rank + 7) / 8 * 8, rot_dim, 0, page};
  out->row_ld = (out->rank_pad + rot_dim + 63) / 64 * 64;
  return check_latent("nf_latent_layout_of", *out);
}

int nf_latent_append(const nf_latent_layout* layout, const void* proj, int ld, int q_col, int kv_col, const float* norm, float eps,
                     const nf_rotation* rot, void* q, void* kv_data, const int32_t* kv_indptr, const int32_t* kv_indices,
                     const int32_t* rev_input_indptr, const int32_t* positions, int rows, int q_rows, nf_stream_t stream) {
  const char* who = "nf_latent_append";
  NF_REQUIRE(layout && rot, "%s: null pointer", who);
  const nf_latent_layout& l = *layout;
  int rc = check_latent(who, l);
  if (rc) return rc;
  NF_REQUIRE(rot->dims >= 0 && rot->dims % 2 == 0 && rot->dims <= l.rot_dim && (rot->dims == 0 || rot->table), "%s: %d of %d dimensions rotated",
             who, rot->dims, l.rot_dim);
  NF_REQUIRE(rows >= 0 && q_col >= 0 && kv_col >= 0 && q_col + l.heads * l.rot_dim <= ld && kv_col + l.kv_rank + l.rot_dim <= ld,
             "%s: columns %d %d do not fit rows of %d", who, q_col, kv_col, ld);
  if (rows == 0) return NF_OK;
  NF_REQUIRE(proj && norm && q && kv_data && kv_indptr && kv_indices && rev_input_indptr && positions, "%s: null pointer", who);
  hipStream_t s = (hipStream_t)stream;
  if (l.dtype == NF_BF16)
    latent_append_kernel<bf16_t><<<rows, 256, 0, s>>>(l, (const bf16_t*)proj, ld, q_col, kv_col, norm, eps, *rot, (bf16_t*)q, (bf16_t*)kv_data,
                                                      kv_indptr, kv_indices, rev_input_indptr, positions, q_rows);
  else
    latent_append_kernel<float><<<rows, 256, 0, s>>>(l, (const float*)proj, ld, q_col, kv_col, norm, eps, *rot, (float*)q, (float*)kv_data,
                                                     kv_indptr, kv_indices, rev_input_indptr, positions, q_rows);
  return check_launch(who);
}

static int check_expand(const char* who, const nf_latent_expand_args* a) {
  NF_REQUIRE(a, "%s: null pointer", who);
  const int rc = check_latent(who, a->layout);
  if (rc) return rc;
  const nf_kv_layout& kv = a->kv;
  NF_REQUIRE(kv.dtype == a->layout.dtype && kv.maps == 1 && kv.heads == a->layout.heads && kv.kv_heads == kv.heads && kv.page == kLatentPage && a->dim_pad > 0 &&
                 a->dim_pad % 8 == 0 && kv.dim == a->dim_pad + a->layout.rot_dim && kv.dim <= 256 && kv.vdim > 0 && kv.vdim % 8 == 0 &&
                 kv.vdim <= 256 && kv.k_pad == (kv.dim + 31) / 32 * 32 && kv.v_pad == (kv.vdim + 15) / 16 * 16,
             "%s: %d heads of %d + %d and %d", who, kv.heads, a->dim_pad, a->layout.rot_dim, kv.vdim);
  NF_REQUIRE(a->max_pages >= 0 && a->max_pages <= 65535 && a->req_begin >= 0 && a->req_end >= a->req_begin, "%s: %d pages of requests %d .. %d", who,
             a->max_pages, a->req_begin, a->req_end);
  NF_REQUIRE(a->max_pages == 0 || (a->kv_data && a->kv_indptr && a->kv_indices), "%s: null pointer", who);
  return NF_OK;
}

int nf_latent_gather(const nf_latent_expand_args* args, nf_stream_t stream) {
  const char* who = "nf_latent_gather";
  const int rc = check_expand(who, args);
  if (rc || args->max_pages == 0) return rc;
  NF_REQUIRE(args->rows && args->page_ids, "%s: null pointer", who);
  if (args->layout.dtype == NF_BF16) latent_gather_kernel<bf16_t><<<args->max_pages, 256, 0, (hipStream_t)stream>>>(*args);
  else latent_gather_kernel<float><<<args->max_pages, 256, 0, (hipStream_t)stream>>>(*args);
  return check_launch(who);
}

int nf_latent_pack(const nf_latent_expand_args* args, nf_stream_t stream) {
  const char* who = "nf_latent_pack";
  const int rc = check_expand(who, args);
  if (rc || args->max_pages == 0) return rc;
  const nf_latent_expand_args& a = *args;
  NF_REQUIRE(a.products && a.pages, "%s: null pointer", who);
  NF_REQUIRE(a.ld % 8 == 0 && a.k_col >= 0 && a.v_col >= 0 && (a.k_col | a.v_col) % 8 == 0 && a.k_col + a.kv.heads * a.dim_pad <= a.ld &&
                 a.v_col + a.kv.heads * a.kv.vdim <= a.ld,
             "%s: columns %d %d do not fit rows of %d", who, a.k_col, a.v_col, a.ld);
  const dim3 grid((unsigned)a.kv.heads, (unsigned)a.max_pages);
  if (a.layout.dtype == NF_BF16) latent_pack_kernel<bf16_t><<<grid, 256, 0, (hipStream_t)stream>>>(a);
  else latent_pack_kernel<float><<<grid, 256, 0, (hipStream_t)stream>>>(a);
  return check_launch(who);
}

int nf_latent_queries(const nf_kv_layout* kv, int dim_pad, const void* proj, int ld, int q_col, int rot_dim, const nf_rotation* rot,
                      const int32_t* positions, void* q, int row_begin, int rows, nf_stream_t stream) {
  const char* who = "nf_latent_queries";
  NF_REQUIRE(kv && rot, "%s: null pointer", who);
  NF_REQUIRE(kv->heads > 0 && dim_pad > 0 && dim_pad % 8 == 0 && rot_dim >= 0 && kv->dim == dim_pad + rot_dim && kv->k_pad == (kv->dim + 31) / 32 * 32 &&
                 ld % 8 == 0 && kv->heads * dim_pad <= ld && q_col >= 0 && q_col + kv->heads * rot_dim <= ld && row_begin >= 0 && rows >= 0,
             "%s: %d heads of %d + %d, column %d of rows of %d", who, kv->heads, dim_pad, rot_dim, q_col, ld);
  NF_REQUIRE(rot->dims >= 0 && rot->dims % 2 == 0 && rot->dims <= rot_dim && (rot->dims == 0 || rot->table), "%s: %d of %d dimensions rotated", who,
             rot->dims, rot_dim);
  if (rows == 0) return NF_OK;
  NF_REQUIRE(proj && positions && q, "%s: null pointer", who);
  hipStream_t s = (hipStream_t)stream;
  if (kv->dtype == NF_BF16)
    latent_queries_kernel<bf16_t><<<rows, 256, 0, s>>>(*kv, dim_pad, (const bf16_t*)proj, ld, q_col, rot_dim, *rot, positions, (bf16_t*)q, row_begin);
  else
    latent_queries_kernel<float><<<rows, 256, 0, s>>>(*kv, dim_pad, (const float*)proj, ld, q_col, rot_dim, *rot, positions, (float*)q, row_begin);
  return check_launch(who);
}

size_t nf_latent_workspace_bytes(const nf_latent_layout* l, int max_rows) {
  if (!l || l->dtype != NF_BF16 || max_rows <= 0) return 0;
  // splits x rows is largest where the tiles alone just do not fill the chip
  const size_t pairs = std::max<size_t>(512 * 16, std::min<size_t>((size_t)max_rows, 256) * l->heads * 2);
  return std::min(pairs, (size_t)max_rows * l->heads * kMaxSplits) * (l->rank_pad + 2) * sizeof(float);
}

int nf_latent_attention(const nf_latent_attention_args* args, nf_stream_t stream) {
  const char* who = "nf_latent_attention";
  NF_REQUIRE(args, "%s: null pointer", who);
  const nf_latent_attention_args& a = *args;
  int rc = check_latent(who, a.layout);
  if (rc) return rc;
  NF_REQUIRE(a.req_num >= 0 && a.req_begin >= 0 && a.max_rows >= 0 && a.row_begin >= 0, "%s: requests %d + %d, rows %d + %d", who, a.req_begin,
             a.req_num, a.row_begin, a.max_rows);
  NF_REQUIRE(!a.decode || a.max_rows == a.req_num, "%s: %d decode requests with %d rows", who, a.req_num, a.max_rows);
  if (a.req_num == 0 || a.max_rows == 0) return NF_OK;
  NF_REQUIRE(a.q && a.out && a.kv_data && a.input_indptr && a.kv_indptr && a.kv_indices && a.rev_input_indptr && a.positions, "%s: null pointer",
             who);
  hipStream_t s = (hipStream_t)stream;
  const nf_latent_layout& l = a.layout;
  // the matrix kernel takes the maximum before it scales
  if (l.dtype == NF_BF16 && a.scale > 0.f && l.row_ld <= 576 && l.rank_pad <= 512) {
    if (l.row_ld == 576 && l.rank_pad == 512) return launch_latent<18, 32, true>(a, s);
    if (l.row_ld <= 192 && l.rank_pad <= 128) return launch_latent<6, 8, false>(a, s);
    if (l.row_ld <= 320 && l.rank_pad <= 256) return launch_latent<10, 16, false>(a, s);
    return launch_latent<18, 32, false>(a, s);
  }
  const dim3 grid((unsigned)a.max_rows, (unsigned)l.heads);
  const bool wide = l.rank_pad > 512;
  if (l.dtype == NF_BF16) {
    if (wide) latent_rows_kernel<bf16_t, kMaxRank / 64><<<grid, 64, 0, s>>>(a);
    else latent_rows_kernel<bf16_t, 8><<<grid, 64, 0, s>>>(a);
  } else {
    if (wide) latent_rows_kernel<float, kMaxRank / 64><<<grid, 64, 0, s>>>(a);
    else latent_rows_kernel<float, 8><<<grid, 64, 0, s>>>(a);
  }
  return check_launch(who);
}

}  // extern "C"
