// Attention of the layer-stack pipeline: short convolution + per-head norm + rotation + query temperature + append
// to the paged cache, and attention over a window or a chunk with kept first positions, capped scores, a sink in the softmax,
// outputs turned back and a gate per head, for any head sizes; also the difference of two attentions of a head over the same values.
//
// bf16 (attn_window_kernel, v_mfma_f32_16x16x32_bf16): S^T = K . Q^T, then O^T = V^T . P^T, per
// (request, kv head, up to 16 of its query heads).  The 16 MFMA columns carry (token, head) pairs.
//   * The rows of the two 16-key score tiles of a 32-key step are assigned so that a lane ends up with
//     8 CONSECUTIVE keys of its column -- row 4g + r of tile b is key 8g + 4b + r -- which is the
//     second product's operand without a permute; V is cached transposed (a value column's 16 positions
//     of a page are contiguous), so its operand is one 16-byte load as well.  Neither goes through LDS.
//   * Softmax weights keep 32 bits: P is multiplied as two bf16 terms, P = hi + lo.
//   * Two maps of a head are two sets of columns beside each other, with keys of their own: a value fragment serves
//     both, and their difference and its norm are taken in fp32 where the sums are.
//   * Only the 32-key steps that hold a visible key are visited: those of the kept first positions,
//     then those of the window.
//   * decode: one token per request, the wavefronts of a workgroup take every n-th step and merge
//     (m, l, O) through LDS.  prefill: every wavefront has NB column blocks of its own and walks their
//     keys; the keys of the next step are requested while the current one is computed.
//   * prefill of the usual head sizes (attn_tile_kernel): the same products, but a workgroup's wavefronts share their
//     keys and values, 32 of them at a time, through a ring of four LDS slots that are filled without registers
//     (buffer_load ... lds), three in flight while one is computed.
// fp32 (attn_rows_kernel): one wavefront per (row, head), every product in 32-bit.
#include <algorithm>
#include <cmath>
#include <type_traits>

#include "layer_common.h"

namespace nf {

constexpr int kPage = 16;
constexpr int kMaxHeadDim = 256;

__host__ __device__ inline size_t kv_page_elements(const nf_kv_layout& kv) {
  return (size_t)kv.kv_heads * kv.page * (kv.maps * kv.k_pad + kv.v_pad);
}
__host__ __device__ inline size_t kv_value_offset(const nf_kv_layout& kv) { return (size_t)kv.kv_heads * kv.maps * kv.page * kv.k_pad; }

// ---------------------------------------------------------------- norm, rotation, append
__device__ __forceinline__ float temperature(const nf_query_temperature& q, int pos) {
  return q.every > 0 ? 1.f + q.coef * logf((float)((pos + 1) / q.every + 1)) : 1.f;
}

// Column c of a row whose columns 2m and 2m + 1 are turned by `way` (1 or -1) times the position; `other`: its pair's other one.
__device__ __forceinline__ float turn_pair(float y, float other, const nf_rotation& rot, int pos, int c, float way) {
  if (c >= rot.dims) return y;
  const float* t = rot.table + (size_t)pos * rot.dims + (c & ~1);
  return y * t[0] + (c & 1 ? way : -way) * other * t[1];
}
// The same of columns c .. c + 3, c a multiple of four.
__device__ __forceinline__ float4_t turn_four(float4_t x, const nf_rotation& rot, int pos, int c, float way) {
  typedef float f32x2_t __attribute__((ext_vector_type(2)));
  if (c >= rot.dims) return x;
  const float* t = rot.table + (size_t)pos * rot.dims + c;
  const f32x2_t a = *reinterpret_cast<const f32x2_t*>(t), b = *reinterpret_cast<const f32x2_t*>(t + (c + 2 < rot.dims ? 2 : 0));
  float4_t y{x[0] * a[0] - way * x[1] * a[1], x[1] * a[0] + way * x[0] * a[1], x[2], x[3]};
  if (c + 2 < rot.dims) {
    y[2] = x[2] * b[0] - way * x[3] * b[1];
    y[3] = x[3] * b[0] + way * x[2] * b[1];
  }
  return y;
}

template <int N>
using Int = std::integral_constant<int, N>;

template <class T>
struct ConvRow;
template <int R, class T>
__device__ __forceinline__ void four_of(const ConvRow<T>* row, int c, const bool* owner, float4_t* y);

// A row of the projections as the short convolution sees it: rows before it, of the batch or of the request's slot.
template <class T>
struct ConvRow {
  const T* proj = nullptr;  // this row
  const T* weight = nullptr;
  T* state = nullptr;       // of the request's slot
  int taps = 0, ld = 0, pos = 0;
  int before = 0;           // rows of the portion ahead of this one
  int place = 0;            // of this row in the state, which is a ring of taps - 1 rows
  bool single = false;      // the request's only row, which leaves the state as well

  __device__ __forceinline__ ConvRow(const nf_short_conv& c, const T* proj_, int ld_, int t, int req, int pos_)
      : proj(proj_ + (size_t)t * ld_), weight((const T*)c.weight), taps(c.taps), ld(ld_), pos(pos_) {
    if (taps < 1) return;
    const int first = c.input_indptr[req];
    before = t - first;
    single = c.input_indptr[req + 1] - first == 1;
    if (taps > 1) {
      state = (T*)c.state + (size_t)c.state_slots[req] * (taps - 1) * ld;
      place = pos % (taps - 1);
    }
  }
  __device__ __forceinline__ ConvRow() {}
  // its value j rows back, j in 0 .. min(taps - 1, pos)
  __device__ __forceinline__ const T* back(int j) const {
    return j <= before ? proj - (size_t)j * ld : state + (size_t)(place - j + (place < j ? taps - 1 : 0)) * ld;
  }
  __device__ __forceinline__ float4_t four(int c, bool owner) const {
    float4_t y;
    four_of<1>(this, c, &owner, &y);
    return y;
  }
  __device__ __forceinline__ float one(int c) const {  // asked for by the owner only
    const T cur = proj[c];
    if (taps < 1) return Act<T>::load(&cur);
    float y = 0.f;
    for (int j = 1; j <= min(taps - 1, pos); ++j) y += Act<T>::load(back(j) + c) * Act<T>::load(weight + (size_t)(taps - 1 - j) * ld + c);
    y += Act<T>::load(&cur) * Act<T>::load(weight + (size_t)(taps - 1) * ld + c);
    if (single && taps > 1) state[(size_t)place * ld + c] = cur;
    return y;
  }
};

// Columns c .. c + 3 of R rows that follow each other, everything requested at once; owner[u]: of the threads that ask for
// them, the one that keeps row u's state.
template <int R, class T>
__device__ __forceinline__ void four_of(const ConvRow<T>* row, int c, const bool* owner, float4_t* y) {
  typedef typename Act<T>::raw4 raw4;
  raw4 cur[R];
#pragma unroll
  for (int u = 0; u < R; ++u) cur[u] = Act<T>::load_raw4(row[u].proj + c);
  const int taps = row[0].taps, ld = row[0].ld;
  if (taps < 1) {
#pragma unroll
    for (int u = 0; u < R; ++u) y[u] = Act<T>::widen4(cur[u]);
    return;
  }
  const float4_t zero{0.f, 0.f, 0.f, 0.f}, last = Act<T>::load4(row[0].weight + (size_t)(taps - 1) * ld + c);
  auto weight = [&](int j) { return Act<T>::load_raw4(row[0].weight + (size_t)(taps - 1 - min(j, taps - 1)) * ld + c); };
  // past the first token or the last tap: the furthest there is again, left out of the sums
  auto before = [&](int u, int j) { return Act<T>::load_raw4(row[u].back(min(j, min(taps - 1, row[u].pos))) + c); };
  constexpr int kAhead = 3;
  if (R > 1 && taps <= kAhead + 1 && row[R - 1].before >= R - 1) {  // all of one portion: every row is read once
    raw4 x[kAhead], w[kAhead];
    float4_t at[R + kAhead], f[kAhead];  // at[kAhead + u]: row u
#pragma unroll
    for (int k = 0; k < kAhead; ++k) w[k] = weight(k + 1);
#pragma unroll
    for (int k = 0; k < kAhead; ++k) x[k] = before(0, k + 1);
#pragma unroll
    for (int k = 0; k < kAhead; ++k) {
      at[kAhead - 1 - k] = k + 1 <= row[0].pos ? Act<T>::widen4(x[k]) : zero;
      f[k] = k + 1 < taps ? Act<T>::widen4(w[k]) : zero;
    }
#pragma unroll
    for (int u = 0; u < R; ++u) at[kAhead + u] = Act<T>::widen4(cur[u]);
#pragma unroll
    for (int u = 0; u < R; ++u) {
      y[u] = zero;
#pragma unroll
      for (int k = 0; k < kAhead; ++k) y[u] += at[kAhead + u - 1 - k] * f[k];
      y[u] += at[kAhead + u] * last;
    }
    return;  // rows of such a portion are not single
  }
#pragma unroll
  for (int u = 0; u < R; ++u) y[u] = zero;
  for (int j0 = 1; j0 < taps; j0 += kAhead) {
    raw4 x[R][kAhead], w[kAhead];
#pragma unroll
    for (int k = 0; k < kAhead; ++k) w[k] = weight(j0 + k);
#pragma unroll
    for (int u = 0; u < R; ++u)
#pragma unroll
      for (int k = 0; k < kAhead; ++k) x[u][k] = before(u, j0 + k);
#pragma unroll
    for (int u = 0; u < R; ++u)
#pragma unroll
      for (int k = 0; k < kAhead; ++k)
        if (j0 + k <= min(taps - 1, row[u].pos)) y[u] += Act<T>::widen4(x[u][k]) * Act<T>::widen4(w[k]);
  }
#pragma unroll
  for (int u = 0; u < R; ++u) {
    y[u] += Act<T>::widen4(cur[u]) * last;
    if (owner[u] && row[u].single && taps > 1) *reinterpret_cast<raw4*>(row[u].state + (size_t)row[u].place * ld + c) = cur[u];
  }
}

// The last rows of every request that brings more than one, as the state of its convolution.  Sixteen bytes a thread.
template <class T>
__global__ __launch_bounds__(256) void conv_state_kernel(const T* __restrict__ proj, int ld, nf_short_conv conv, const int32_t* __restrict__ positions,
                                                         int req_begin) {
  const int req = req_begin + blockIdx.x, first = conv.input_indptr[req], end = conv.input_indptr[req + 1];
  const int c = (blockIdx.y * 256 + threadIdx.x) * (16 / (int)sizeof(T)), keep = conv.taps - 1;
  if (end - first < 2 || c >= ld) return;
  T* state = (T*)conv.state + (size_t)conv.state_slots[req] * keep * ld;
  for (int t = max(first, end - keep); t < end; ++t)
    *reinterpret_cast<u32x4*>(state + (size_t)((positions[first] + t - first) % keep) * ld + c) = *reinterpret_cast<const u32x4*>(proj + (size_t)t * ld + c);
}

// One wavefront per (row, head): query heads, then key heads, then value heads.
template <class T>
__global__ __launch_bounds__(256) void qkv_append_kernel(nf_kv_layout kv, const T* __restrict__ proj, int ld, int q_col,
                                                         int k_col, int v_col, const float* __restrict__ q_norm,
                                                         const float* __restrict__ k_norm, float eps, nf_rotation rot,
                                                         nf_query_temperature q_temp, nf_value_form vform, nf_short_conv conv, T* __restrict__ q_out, T* __restrict__ kv_data,
                                                         const int32_t* __restrict__ kv_indptr,
                                                         const int32_t* __restrict__ kv_indices,
                                                         const int32_t* __restrict__ rev_input_indptr,
                                                         const int32_t* __restrict__ positions) {
  __shared__ float row_buf[4][kMaxHeadDim];
  const int t = blockIdx.x, lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int job = blockIdx.y * 4 + wave;
  const int H = kv.heads * kv.maps, G = kv.kv_heads * kv.maps, VG = kv.kv_heads;
  const int pos = positions[t], req = rev_input_indptr[t];
  const ConvRow<T> row(conv, proj, ld, t, req, pos);
  T* page = nullptr;
  int entry = 0;
  if (job >= H && job < H + G + VG) {
    page = kv_data + (size_t)kv_indices[kv_indptr[req] + pos / kPage] * kv_page_elements(kv);
    entry = pos % kPage;
  }
  const bool is_qk = job < H + G;
  if (is_qk) {
    const bool is_q = job < H;
    const int head = is_q ? job : job - H;
    const int col = (is_q ? q_col : k_col) + head * kv.dim;
    const float* w = is_q ? q_norm : k_norm;
    float v[kMaxHeadDim / 64];
    float sq = 0.f;
#pragma unroll
    for (int i = 0; i < kMaxHeadDim / 64; ++i) {
      const int c = i * 64 + lane;
      v[i] = c < kv.dim ? row.one(col + c) : 0.f;
      sq += v[i] * v[i];
    }
    if (w) {
      const float inv = 1.f / sqrtf(wave_sum(sq) / (float)kv.dim + eps);
#pragma unroll
      for (int i = 0; i < kMaxHeadDim / 64; ++i) {
        const int c = i * 64 + lane;
        if (c < kv.dim) v[i] = v[i] * inv * w[c];
      }
    }
#pragma unroll
    for (int i = 0; i < kMaxHeadDim / 64; ++i) row_buf[wave][i * 64 + lane] = v[i];
  }
  __syncthreads();  // a lane's rotation partner is another lane's element
  if (is_qk) {
    const bool is_q = job < H;
    const int head = is_q ? job : job - H;
    T* dst = is_q ? q_out + ((size_t)t * H + head) * kv.k_pad : page + ((size_t)head * kPage + entry) * kv.k_pad;
    const int half = rot.dims / 2;
    const float temp = is_q ? temperature(q_temp, pos) : 1.f;
#pragma unroll
    for (int i = 0; i < kMaxHeadDim / 64; ++i) {
      const int c = i * 64 + lane;
      if (c >= kv.k_pad) continue;
      float y = row_buf[wave][c];  // zero past dim
      if (c < 2 * half) {
        const int f = rot.interleaved ? c >> 1 : (c < half ? c : c - half);
        const bool first = rot.interleaved ? !(c & 1) : c < half;
        const float other = row_buf[wave][rot.interleaved ? c ^ 1 : (first ? c + half : c - half)];
        const float cs = rot.table[((size_t)pos * half + f) * 2], sn = rot.table[((size_t)pos * half + f) * 2 + 1];
        y = first ? y * cs - other * sn : y * cs + other * sn;
      }
      Act<T>::store(dst + c, y * temp);
    }
  } else if (job < H + G + VG) {
    const int head = job - H - G;
    T* dst = page + kv_value_offset(kv) + (size_t)head * kv.v_pad * kPage + entry;
    float v[kMaxHeadDim / 64];
    float sq = 0.f;
#pragma unroll
    for (int i = 0; i < kMaxHeadDim / 64; ++i) {
      const int c = i * 64 + lane;
      v[i] = c < kv.vdim ? row.one(v_col + head * kv.vdim + c) : 0.f;
      sq += v[i] * v[i];
    }
    const float inv = vform.norm ? 1.f / sqrtf(wave_sum(sq) / (float)kv.vdim + eps) : 1.f;
#pragma unroll
    for (int i = 0; i < kMaxHeadDim / 64; ++i) {
      const int c = i * 64 + lane;
      float y = v[i] * inv;
      if (vform.rot.dims > 0) y = turn_pair(y, __shfl_xor(y, 1, 64), vform.rot, pos, c, 1.f);
      if (c < kv.v_pad) Act<T>::store(dst + (size_t)c * kPage, y);
    }
  }
}

// The same for sizes and columns that are multiples of four, which is what models have.  A workgroup takes R rows of 16
// heads, 16 lanes a head, kVec groups of four elements a lane, so that everything about a row is the same in all its
// lanes.  Of many rows, values are turned through LDS, 16 rows of a head at a time, so that the transposed cache is
// written four positions at once where four rows are an aligned run of one page; of few (value_blocks = 0) value heads
// are taken like the others.
template <class T, int kVec, int R, bool kConv>
__global__ __launch_bounds__(256, kVec <= 2 ? 8 : 5) void qkv_append4_kernel(nf_kv_layout kv, const T* __restrict__ proj, int ld, int q_col,
                                                          int k_col, int v_col, const float* __restrict__ q_norm,
                                                          const float* __restrict__ k_norm, float eps, nf_rotation rot,
                                                          nf_query_temperature q_temp, nf_value_form vform, nf_short_conv conv, T* __restrict__ q_out, T* __restrict__ kv_data,
                                                          const int32_t* __restrict__ kv_indptr,
                                                          const int32_t* __restrict__ kv_indices,
                                                          const int32_t* __restrict__ rev_input_indptr,
                                                          const int32_t* __restrict__ positions, int rows, int value_blocks) {
  __shared__ __attribute__((aligned(16))) float buf[kMaxHeadDim * 17];
  if constexpr (!kConv) conv.taps = 0;  // its code is left out
  const int H = kv.heads * kv.maps, G = kv.kv_heads * kv.maps, VG = kv.kv_heads, tid = threadIdx.x;
  if ((int)blockIdx.x >= value_blocks) {
    const int jobs = H + G + (value_blocks > 0 ? 0 : VG), head_blocks = (jobs + 15) / 16, block = blockIdx.x - value_blocks;
    const int t0 = block / head_blocks * R, l = tid & 15, job = block % head_blocks * 16 + (tid >> 4);
    const bool live = job < jobs;
    const int head = live ? job : 0;
    const bool is_q = head < H, is_v = head >= H + G;
    const int dim = is_v ? kv.vdim : kv.dim;
    const int col = is_q ? q_col + head * dim : is_v ? v_col + (head - H - G) * dim : k_col + (head - H) * dim;
    const float* w = is_q ? q_norm : is_v ? nullptr : k_norm;
    float* mine = buf + (tid >> 4) * (kVec * 64);
    const int half = is_v ? 0 : rot.dims / 2;
    ConvRow<T> row[R];
    T* dst[R];
    bool keep[R];
#pragma unroll
    for (int u = 0; u < R; ++u) {
      const int t = min(t0 + u, rows - 1), pos = positions[t], req = rev_input_indptr[t];
      row[u] = ConvRow<T>(conv, proj, ld, t, req, pos);
      keep[u] = live && t0 + u < rows;
      T* page = kv_data + (size_t)kv_indices[kv_indptr[req] + pos / kPage] * kv_page_elements(kv);
      dst[u] = is_q   ? q_out + ((size_t)t * H + head) * kv.k_pad
               : is_v ? page + kv_value_offset(kv) + (size_t)(head - H - G) * kv.v_pad * kPage + pos % kPage
                      : page + ((size_t)(head - H) * kPage + pos % kPage) * kv.k_pad;
    }
    float4_t v[kVec][R];
#pragma unroll
    for (int i = 0; i < kVec; ++i) {
      const int c = (i * 16 + l) * 4;
#pragma unroll
      for (int u = 0; u < R; ++u) v[i][u] = float4_t{0.f, 0.f, 0.f, 0.f};
      if (c < dim) four_of<R>(row, col + c, keep, v[i]);
    }
    if (q_norm || k_norm || vform.norm) {  // asked by the whole workgroup: the sums are over lanes
#pragma unroll
      for (int u = 0; u < R; ++u) {
        float sq = 0.f;
#pragma unroll
        for (int i = 0; i < kVec; ++i)
#pragma unroll
          for (int e = 0; e < 4; ++e) sq += v[i][u][e] * v[i][u][e];
#pragma unroll
        for (int m = 8; m > 0; m >>= 1) sq += __shfl_xor(sq, m, 64);
        const float inv = 1.f / sqrtf(sq / (float)dim + eps);
        if (w) {
#pragma unroll
          for (int i = 0; i < kVec; ++i) {
            const int c = (i * 16 + l) * 4;
            if (c < dim) v[i][u] = v[i][u] * inv * *reinterpret_cast<const float4_t*>(w + c);
          }
        } else if (is_v && vform.norm) {
#pragma unroll
          for (int i = 0; i < kVec; ++i) v[i][u] *= inv;
        }
      }
    }
#pragma unroll
    for (int u = 0; u < R; ++u) {
      const float temp = is_q ? temperature(q_temp, row[u].pos) : 1.f;
      const float* tab = rot.table + (size_t)row[u].pos * half * 2;
      if (!rot.interleaved) {  // a lane's partners are in its own wavefront
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
        __builtin_amdgcn_wave_barrier();
#pragma unroll
        for (int i = 0; i < kVec; ++i) *reinterpret_cast<float4_t*>(mine + (i * 16 + l) * 4) = v[i][u];
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
        __builtin_amdgcn_wave_barrier();
      }
#pragma unroll
      for (int i = 0; i < kVec; ++i) {
        const int c = (i * 16 + l) * 4;
        const float4_t x = v[i][u];
        float4_t y = x;
        if (c < 2 * half) {
          if (rot.interleaved) {
            const float4_t cs = *reinterpret_cast<const float4_t*>(tab + c);  // cos, sin of pair c / 2, then of the next
            y = float4_t{x[0] * cs[0] - x[1] * cs[1], x[1] * cs[0] + x[0] * cs[1], x[2] * cs[2] - x[3] * cs[3], x[3] * cs[2] + x[2] * cs[3]};
          } else {
            const bool first = c < half;
            const int f = first ? c : c - half;
            const float4_t other = *reinterpret_cast<const float4_t*>(mine + (first ? c + half : f));
            const float4_t a = *reinterpret_cast<const float4_t*>(tab + 2 * f), b = *reinterpret_cast<const float4_t*>(tab + 2 * f + 4);
            const float4_t cs{a[0], a[2], b[0], b[2]}, sn{a[1], a[3], b[1], b[3]};
            y = first ? x * cs - other * sn : x * cs + other * sn;
          }
        }
        y = y * temp;
        if (is_v) {
          if (vform.rot.dims > 0) y = turn_four(y, vform.rot, row[u].pos, c, 1.f);
          if (keep[u] && c < kv.v_pad)
#pragma unroll
            for (int e = 0; e < 4; ++e) Act<T>::store(dst[u] + (size_t)(c + e) * kPage, y[e]);
        } else if (keep[u] && c < kv.k_pad) {
          Act<T>::store4(dst[u] + c, y);
        }
      }
    }
    return;
  }
  __shared__ long long row_page[16];  // element offset of the row's page, and its entry
  __shared__ int row_entry[16];
  const int head = blockIdx.x % VG, row0 = blockIdx.x / VG * 16;
  if (tid < 16) {
    const int t = min(row0 + tid, rows - 1), pos = positions[t];
    row_page[tid] = (long long)kv_indices[kv_indptr[rev_input_indptr[t]] + pos / kPage] * (long long)kv_page_elements(kv);
    row_entry[tid] = row0 + tid < rows ? pos % kPage : -1;
  }
  const int r = tid >> 4, t = min(row0 + r, rows - 1);
  const ConvRow<T> row(conv, proj, ld, t, rev_input_indptr[t], positions[t]);
  float inv = 1.f;
  if (vform.norm) {  // the row's 16 lanes are of one wavefront; what they read here they read again below, from the cache
    float sq = 0.f;
    for (int c = (tid & 15) * 4; c < kv.vdim; c += 64) {
      const float4_t v = row.four(v_col + head * kv.vdim + c, false);
      sq += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
    }
#pragma unroll
    for (int m = 8; m > 0; m >>= 1) sq += __shfl_xor(sq, m, 64);
    inv = 1.f / sqrtf(sq / (float)kv.vdim + eps);
  }
  for (int c = (tid & 15) * 4; c < kv.v_pad; c += 64) {
    float4_t v{0.f, 0.f, 0.f, 0.f};
    if (c < kv.vdim) v = row.four(v_col + head * kv.vdim + c, row0 + r < rows) * inv;
    if (vform.rot.dims > 0) v = turn_four(v, vform.rot, row.pos, c, 1.f);
#pragma unroll
    for (int e = 0; e < 4; ++e) buf[(c + e) * 17 + r] = v[e];
  }
  __syncthreads();
  T* base = kv_data + kv_value_offset(kv) + (size_t)head * kv.v_pad * kPage;
  for (int e = tid; e < kv.v_pad * 4; e += 256) {
    const int c = e >> 2, r0 = (e & 3) * 4, en = row_entry[r0];
    const float* v = buf + c * 17 + r0;
    if (en >= 0 && en % 4 == 0 && row_entry[r0 + 3] == en + 3 && row_page[r0] == row_page[r0 + 3]) {
      // rows of one request are consecutive positions, so the two in between belong to the run as well
      Act<T>::store4(base + row_page[r0] + (size_t)c * kPage + en, float4_t{v[0], v[1], v[2], v[3]});
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (row_entry[r0 + i] >= 0) Act<T>::store(base + row_page[r0 + i] + (size_t)c * kPage + row_entry[r0 + i], v[i]);
    }
  }
}

// ---------------------------------------------------------------- which 32-key (or 64-key) steps are visited
struct StepRange {
  int head, skip_to, total;  // steps [0, head), then [skip_to, ...): `total` of both
  __device__ __forceinline__ int at(int i) const { return i < head ? i : skip_to + i - head; }
};
// The first position that one at p sees, the kept first ones aside; it does not fall as p grows.
__device__ __forceinline__ int first_seen(const nf_window_attention_args& a, int p) {
  const int lo = a.window > 0 ? p - a.window + 1 : 0;
  return a.chunk > 0 ? max(lo, p - p % a.chunk) : lo;
}
// The steps of `width` keys in which a token at a position in [p0, p1] sees a key.
__device__ __forceinline__ StepRange visible_steps(const nf_window_attention_args& a, int p0, int p1, int width) {
  const int end = p1 / width + 1;
  const int lo = first_seen(a, p0);
  if (lo <= 0) return {0, 0, end};
  const int kept = a.keep_first > p1 + 1 ? p1 + 1 : a.keep_first;
  const int head = (kept + width - 1) / width;
  int skip_to = lo > 0 ? lo / width : 0;
  if (skip_to < head) skip_to = head;
  return {head, skip_to, head + (end > skip_to ? end - skip_to : 0)};
}

// lo: first_seen of p
__device__ __forceinline__ bool sees(int p, int lo, int j, int keep_first) { return j <= p && (j >= lo || j < keep_first); }

// What a head's output is multiplied by in the end.
template <class T>
__device__ __forceinline__ float head_factor(const nf_window_attention_args& a, int row, int h) {
  return a.gate ? a.out_scale * sigmoid<T>(Act<T>::load((const T*)a.gate + (size_t)row * a.gate_ld + h)) : a.out_scale;
}

// Scores brought within +-softcap, in the exponent's units (base 2): softcap * tanh(s * scale / softcap) * log2 e, with
// tanh x = 1 - 2 / (1 + e^2x).  Without a cap they are left alone and `scale` is still to be applied.
struct ScoreCap {
  float before, limit, scale;
  __device__ __forceinline__ explicit ScoreCap(const nf_window_attention_args& a) {
    constexpr float log2e = 1.44269504088896340736f;
    limit = a.softcap > 0.f ? a.softcap * log2e : 0.f;
    before = a.softcap > 0.f ? 2.f * log2e * a.scale / a.softcap : 0.f;
    scale = a.softcap > 0.f ? 1.f : a.scale * log2e;
  }
  __device__ __forceinline__ void apply(float4_t& s) const {
#pragma unroll
    for (int r = 0; r < 4; ++r) s[r] = fmaf(-2.f * limit, __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(s[r] * before)), limit);
  }
};

// ---------------------------------------------------------------- fp32
template <class T>
__global__ __launch_bounds__(64) void attn_rows_kernel(nf_window_attention_args a) {
  __shared__ __attribute__((aligned(16))) float sq[kMaxHeadDim];
  __shared__ float sp[64];
  const nf_kv_layout kv = a.kv;
  const int lane = threadIdx.x, t = a.row_begin + blockIdx.x, h = blockIdx.y;
  const int req = a.rev_input_indptr[t], p = a.positions[t];
  const int g = h / (kv.heads / kv.kv_heads);
  const T* pool = (const T*)a.kv_data;
  const size_t page_elems = kv_page_elements(kv);
  const int32_t* pages = a.kv_indices + a.kv_indptr[req];
  const StepRange steps = visible_steps(a, p, p, 64);
  const int seen_from = first_seen(a, p);
  float out_row[kMaxHeadDim / 64] = {};
  for (int map = 0; map < kv.maps; ++map) {
    const T* q = (const T*)a.q + (((size_t)t * kv.heads + h) * kv.maps + map) * kv.k_pad;
    __syncthreads();
    for (int c = lane; c < kv.k_pad; c += 64) sq[c] = Act<T>::load(q + c);
    __syncthreads();
    float m = a.sink ? a.sink[h] : -1e30f;
    float l = 0.f;  // this lane's part of the denominator
    float o[kMaxHeadDim / 64] = {};
    for (int i = 0; i < steps.total; ++i) {
      const int base = steps.at(i) * 64, j = base + lane;
      const bool see = sees(p, seen_from, j, a.keep_first);
      float s = -INFINITY;
      if (see) {
        const T* k = pool + (size_t)pages[j / kPage] * page_elems + (((size_t)g * kv.maps + map) * kPage + j % kPage) * kv.k_pad;
        float dot = 0.f;
        for (int c = 0; c < kv.k_pad; c += 4) {
          const float4_t kk = Act<T>::load4(k + c), qq = *reinterpret_cast<const float4_t*>(sq + c);
          dot += kk[0] * qq[0] + kk[1] * qq[1] + kk[2] * qq[2] + kk[3] * qq[3];
        }
        s = dot * a.scale;
        if (a.softcap > 0.f) s = a.softcap * tanhf(s / a.softcap);
      }
      float mx = s;
#pragma unroll
      for (int d = 32; d > 0; d >>= 1) mx = fmaxf(mx, __shfl_xor(mx, d, 64));
      const float m_new = fmaxf(m, mx), alpha = expf(m - m_new);
      const float w = see ? expf(s - m_new) : 0.f;
      m = m_new;
      l = l * alpha + w;
      __syncthreads();
      sp[lane] = w;
      __syncthreads();
#pragma unroll
      for (int e = 0; e < kMaxHeadDim / 64; ++e) o[e] *= alpha;
      const int n_pages = min(4, (p - base) / kPage + 1);
      for (int b = 0; b < n_pages; ++b) {
        const T* v = pool + (size_t)pages[base / kPage + b] * page_elems + kv_value_offset(kv) + (size_t)g * kv.v_pad * kPage;
#pragma unroll
        for (int e = 0; e < kMaxHeadDim / 64; ++e) {
          const int c = e * 64 + lane;
          if (c >= kv.v_pad) break;
#pragma unroll
          for (int r = 0; r < kPage; r += 4) {
            const float4_t vv = Act<T>::load4(v + (size_t)c * kPage + r);
#pragma unroll
            for (int x = 0; x < 4; ++x) {
              const float wt = sp[b * kPage + r + x];
              if (wt != 0.f) o[e] += wt * vv[x];  // an entry past the sequence may hold anything
            }
          }
        }
      }
    }
    l = wave_sum(l);
    if (a.sink) l += expf(a.sink[h] - m);
    const float part = (map == 0 ? 1.f : -a.map_weight) / l;
#pragma unroll
    for (int e = 0; e < kMaxHeadDim / 64; ++e) out_row[e] += o[e] * part;
  }
  float factor = head_factor<T>(a, t, h);
  if (a.head_norm) {
    float sum = 0.f;
#pragma unroll
    for (int e = 0; e < kMaxHeadDim / 64; ++e)
      if (e * 64 + lane < kv.vdim) sum += out_row[e] * out_row[e];
    factor /= sqrtf(wave_sum(sum) / (float)kv.vdim + a.head_eps);
  }
  T* out = (T*)a.out + (size_t)t * a.out_ld + a.out_col + (size_t)h * kv.vdim;
#pragma unroll
  for (int e = 0; e < kMaxHeadDim / 64; ++e) {
    const int c = e * 64 + lane;
    if (a.out_rot.dims > 0) out_row[e] = turn_pair(out_row[e], __shfl_xor(out_row[e], 1, 64), a.out_rot, p, c, -1.f);
    if (c < kv.vdim) Act<T>::store(out + c, out_row[e] * factor);
  }
}

// ---------------------------------------------------------------- bf16
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
union B8 {
  u32x4 u;
  bf16x8_t b;
  uint32_t w[4];
};

template <bool kStream>
__device__ __forceinline__ u32x4 load_cache(const bf16_t* p) {
  typedef uint32_t v4 __attribute__((ext_vector_type(4)));
  if constexpr (kStream) {  // decode reads every cached byte once
    const v4 x = __builtin_nontemporal_load(reinterpret_cast<const v4*>(p));
    return u32x4{x.x, x.y, x.z, x.w};
  } else {
    return *reinterpret_cast<const u32x4*>(p);
  }
}

// What the lanes of a column (those with the same l16) hold of its output in the end, from the sums of its maps; `o` and `l`
// hold kMaps entries.  The value columns are i * 16 + g * 4 ..
template <int kMaps, int VD>
__device__ __forceinline__ void finish_column(const nf_window_attention_args& a, float4_t (*o)[VD], const float* m, const float* l, int row, int pos, int h, int g) {
  float den = l[0], f = 1.f;
  if (a.sink) {
    const float snk = a.sink[h] * 1.44269504088896340736f, mm = fmaxf(m[0], snk);
    f = __builtin_amdgcn_exp2f(m[0] - mm);
    den = den * f + __builtin_amdgcn_exp2f(snk - mm);
  }
  float factor = head_factor<bf16_t>(a, row, h), first = f / den;
  if constexpr (kMaps == 2) {
    const float second = a.map_weight / l[1];
#pragma unroll
    for (int i = 0; i < VD; ++i) o[0][i] = o[0][i] * first - o[1][i] * second;
    first = 1.f;
  }
  if (a.head_norm) {
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < VD; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (i * 16 + g * 4 + r < a.kv.vdim) sum += o[0][i][r] * o[0][i][r];
    factor /= sqrtf(sum_over_lane_groups(sum) * first * first / (float)a.kv.vdim + a.head_eps);
  }
#pragma unroll
  for (int i = 0; i < VD; ++i) o[0][i] *= first * factor;
  if (a.out_rot.dims > 0)
#pragma unroll
    for (int i = 0; i < VD; ++i) o[0][i] = turn_four(o[0][i], a.out_rot, pos, i * 16 + g * 4, -1.f);
}

// KD: 32-wide pieces of k_pad, VD: 16-wide pieces of v_pad (both upper bounds), NB: column blocks per
// wavefront.  gs: query heads of a kv head in one workgroup (at most 16).
constexpr int window_threads(int kMaps, int VD) { return kMaps == 2 && VD > 8 ? 256 : 512; }
template <int KD, int VD, int NB, int kMaps, bool kDecode>
__global__ __launch_bounds__(window_threads(kMaps, VD)) void attn_window_kernel(nf_window_attention_args a, int gs, int chunks, int tile_tokens) {
  extern __shared__ __attribute__((aligned(16))) float merge_lds[];
  const nf_kv_layout kv = a.kv;
  const int lane = threadIdx.x & 63, l16 = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int waves = blockDim.x >> 6;
  const int group = kv.heads / kv.kv_heads;
  const int kvh = blockIdx.y / chunks, h0 = (blockIdx.y % chunks) * gs;  // this workgroup's heads: kvh * group + h0 ...
  const int heads = min(gs, group - h0);
  const int tpb = 16 / gs;  // tokens per column block

  int req, row0, tok0, len;  // request, its first row, this wavefront's first token in it, its rows
  if constexpr (kDecode) {
    req = a.req_begin + blockIdx.x;
    row0 = a.input_indptr[req];
    tok0 = 0;
    len = 1;
  } else {
    int tile = blockIdx.x;
    req = -1;
    for (int r = a.req_begin; r < a.req_begin + a.req_num; ++r) {
      const int n = (a.input_indptr[r + 1] - a.input_indptr[r] + tile_tokens - 1) / tile_tokens;
      if (tile < n) {
        req = r;
        tile = n - 1 - tile;  // the tiles that see most keys start first
        break;
      }
      tile -= n;
    }
    if (req < 0) return;
    row0 = a.input_indptr[req];
    len = a.input_indptr[req + 1] - row0;
    tok0 = tile * tile_tokens + wave * NB * tpb;
    if (tok0 >= len) return;
  }

  constexpr int NC = NB * kMaps;  // sets of columns: a block's maps side by side
  int pos[NB], lo_key[NB], row[NB];
  bool live[NB];
  B8 qf[NC][KD];
  const int kd = kv.k_pad / 32, vd = kv.v_pad / 16;
#pragma unroll
  for (int n = 0; n < NB; ++n) {
    const int tok = kDecode ? 0 : tok0 + n * tpb + l16 / gs, hc = l16 % gs;
    live[n] = (kDecode ? l16 < heads : l16 < tpb * gs && tok < len && hc < heads);
    row[n] = row0 + (live[n] ? tok : (kDecode ? 0 : tok0));
    pos[n] = a.positions[row[n]];
    lo_key[n] = first_seen(a, pos[n]);
    const bf16_t* q = (const bf16_t*)a.q + ((size_t)row[n] * kv.heads + kvh * group + h0 + (live[n] ? hc : 0)) * kMaps * kv.k_pad + g * 8;
#pragma unroll
    for (int x = 0; x < kMaps; ++x)
#pragma unroll
      for (int j = 0; j < KD; ++j)
        qf[n * kMaps + x][j].u = live[n] && j < kd ? *reinterpret_cast<const u32x4*>(q + x * kv.k_pad + j * 32) : u32x4{0, 0, 0, 0};
  }
  const int p0 = a.positions[row0 + tok0];
  const int p1 = kDecode ? p0 : p0 + min(NB * tpb, len - tok0) - 1;
  const StepRange steps = visible_steps(a, p0, p1, 32);
  const int all_from = first_seen(a, p1);  // every token sees the keys from here to its own

  const size_t page_elems = kv_page_elements(kv);
  const int32_t* pages = a.kv_indices + a.kv_indptr[req];
  const int last_page = p1 / kPage;
  const bf16_t* pool = (const bf16_t*)a.kv_data;
  // this lane's pieces inside a page: K rows of tile b (b = 0, 1), V column piece
  const int key = 8 * (l16 >> 2) + (l16 & 3);  // of tile 0 in the step; tile 1: + 4
  const int kpg = key >> 4;                    // its page of the step's two (tile 1's is the same)
  const size_t k_off = ((size_t)kvh * kMaps * kPage + (key & 15)) * kv.k_pad + g * 8;
  const size_t v_off = kv_value_offset(kv) + ((size_t)kvh * kv.v_pad + l16) * kPage + (g & 1) * 8;
  const int vpg = g >> 1;

  float4_t o[NC][VD];
  float m[NC], l[NC];
#pragma unroll
  for (int n = 0; n < NC; ++n) {
    m[n] = -1e30f;
    l[n] = 0.f;
#pragma unroll
    for (int i = 0; i < VD; ++i) o[n][i] = float4_t{0.f, 0.f, 0.f, 0.f};
  }
  const ScoreCap cap(a);
  const float scale2 = cap.scale;

  // page ids are read a step before the loads that need them
  auto page_id = [&](int it, int which) {
    const int idx = steps.at(it) * 2 + which;
    return pages[idx < last_page ? idx : last_page];  // past the last page the keys are no one's: read something mapped
  };
  B8 kf[kMaps][2][KD];
  auto load_k = [&](int id) {
    const bf16_t* k = pool + (size_t)id * page_elems + k_off;
#pragma unroll
    for (int x = 0; x < kMaps; ++x)
#pragma unroll
      for (int j = 0; j < KD; ++j)
        if (j < kd) {
          kf[x][0][j].u = load_cache<kDecode>(k + (size_t)(x * kPage) * kv.k_pad + j * 32);
          kf[x][1][j].u = load_cache<kDecode>(k + (size_t)(x * kPage + 4) * kv.k_pad + j * 32);
        }
  };
  const int first = kDecode ? wave : 0, stride = kDecode ? waves : 1;
  if (first >= steps.total && !kDecode) return;
  const int final_it = steps.total - 1;
  int k_id = page_id(min(first, final_it), kpg), v_id = page_id(min(first, final_it), vpg);
  load_k(k_id);
  k_id = page_id(min(first + stride, final_it), kpg);
  for (int it = first; it < steps.total; it += stride) {
    const int step = steps.at(it), base = step * 32;
    // V of this step, then (after the scores) K of the next: in flight while the softmax runs
    B8 vf[VD];
    const bf16_t* v = pool + (size_t)v_id * page_elems + v_off;
#pragma unroll
    for (int i = 0; i < VD; ++i)
      if (i < vd) vf[i].u = load_cache<kDecode>(v + (size_t)i * 16 * kPage);
    const int next_k_id = page_id(min(it + 2 * stride, final_it), kpg);
    v_id = page_id(min(it + stride, final_it), vpg);
    float4_t s[NC][2];
#pragma unroll
    for (int n = 0; n < NC; ++n)
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        s[n][b] = float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < KD; ++j)
          if (j < kd) s[n][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[n % kMaps][b][j].b, qf[n][j].b, s[n][b], 0, 0, 0);
        if (cap.limit > 0.f) cap.apply(s[n][b]);
      }
    if (it + stride < steps.total) load_k(k_id);
    k_id = next_k_id;
    const bool whole = base + 31 <= p0 && (base >= all_from || base + 31 < a.keep_first);
#pragma unroll
    for (int n = 0; n < NC; ++n) {
      const int j0 = base + 8 * g;
      float mx = -1e30f;
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          if (!whole && !sees(pos[n / kMaps], lo_key[n / kMaps], j0 + 4 * b + r, a.keep_first)) s[n][b][r] = -INFINITY;
          mx = fmaxf(mx, s[n][b][r]);
        }
      mx = mx > -1e30f ? mx * scale2 : mx;
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      // brought to a new maximum only when it has grown by 2^8: weights up to 256 cost nothing in fp32
      if (__any(mx > m[n] + 8.f)) {
        const float m_new = fmaxf(m[n], mx), alpha = __builtin_amdgcn_exp2f(m[n] - m_new);
        m[n] = m_new;
        l[n] *= alpha;
#pragma unroll
        for (int i = 0; i < VD; ++i) o[n][i] *= alpha;
      }
      B8 hi, lo;
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int r = 0; r < 4; r += 2) {
          const float w0 = __builtin_amdgcn_exp2f(fmaf(s[n][b][r], scale2, -m[n]));
          const float w1 = __builtin_amdgcn_exp2f(fmaf(s[n][b][r + 1], scale2, -m[n]));
          l[n] += w0 + w1;
          const uint32_t h2 = f32_to_bf16_pair(w0, w1);
          hi.w[b * 2 + r / 2] = h2;
          lo.w[b * 2 + r / 2] = f32_to_bf16_pair(w0 - __uint_as_float(h2 << 16), w1 - __uint_as_float(h2 & 0xffff0000u));
        }
#pragma unroll
      for (int i = 0; i < VD; ++i)
        if (i < vd) {
          o[n][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[i].b, hi.b, o[n][i], 0, 0, 0);
          o[n][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[i].b, lo.b, o[n][i], 0, 0, 0);
        }
    }
  }

  bf16_t* out = (bf16_t*)a.out;
#pragma unroll
  for (int n = 0; n < NC; ++n) {
    l[n] += __shfl_xor(l[n], 16, 64);
    l[n] += __shfl_xor(l[n], 32, 64);
  }
  if constexpr (kDecode) {
    // merge the wavefronts: m and l of [wave][map][16 columns], O of [wave][map][heads][v_pad]
    float* sm = merge_lds;
    float* sl = sm + waves * kMaps * 16;
    float* so = sl + waves * kMaps * 16;
#pragma unroll
    for (int x = 0; x < kMaps; ++x) {
      if (g == 0) {
        sm[(wave * kMaps + x) * 16 + l16] = m[x];
        sl[(wave * kMaps + x) * 16 + l16] = l[x];
      }
      if (l16 < heads)
#pragma unroll
        for (int i = 0; i < VD; ++i)
          if (i < vd) *reinterpret_cast<float4_t*>(so + ((size_t)(wave * kMaps + x) * gs + l16) * kv.v_pad + i * 16 + g * 4) = o[x][i];
    }
    __syncthreads();
    bf16_t* dst = out + (size_t)row0 * a.out_ld + a.out_col + (size_t)(kvh * group + h0) * kv.vdim;
    for (int e = threadIdx.x; e < heads * kv.vdim; e += blockDim.x) {
      const int hc = e / kv.vdim, c = e % kv.vdim;
      const int h = kvh * group + h0 + hc;
      float v = 0.f;
#pragma unroll
      for (int x = 0; x < kMaps; ++x) {
        const float snk = a.sink ? a.sink[h] * 1.44269504088896340736f : -1e30f;
        float mm = snk;
        for (int w = 0; w < waves; ++w) mm = fmaxf(mm, sm[(w * kMaps + x) * 16 + hc]);
        float den = a.sink ? __builtin_amdgcn_exp2f(snk - mm) : 0.f, acc = 0.f;
        for (int w = 0; w < waves; ++w) {
          const float f = __builtin_amdgcn_exp2f(sm[(w * kMaps + x) * 16 + hc] - mm);
          den += sl[(w * kMaps + x) * 16 + hc] * f;
          acc += so[((size_t)(w * kMaps + x) * gs + hc) * kv.v_pad + c] * f;
        }
        v += acc * ((x == 0 ? 1.f : -a.map_weight) / den);
      }
      if (a.out_rot.dims > 0) v = turn_pair(v, __shfl_xor(v, 1, 64), a.out_rot, p0, c, -1.f);  // heads of an even size: a pair's threads are neighbours
      if (a.head_norm) so[(size_t)hc * kv.v_pad + c] = v;  // read by this thread alone until now
      else Act<bf16_t>::store(dst + e, v * head_factor<bf16_t>(a, row0, h));
    }
    if (!a.head_norm) return;
    __syncthreads();
    for (int hc = wave; hc < heads; hc += waves) {
      const float* v = so + (size_t)hc * kv.v_pad;
      float sum = 0.f;
      for (int c = lane; c < kv.vdim; c += 64) sum += v[c] * v[c];
      const float f = head_factor<bf16_t>(a, row0, kvh * group + h0 + hc) / sqrtf(wave_sum(sum) / (float)kv.vdim + a.head_eps);
      for (int c = lane; c < kv.vdim; c += 64) Act<bf16_t>::store(dst + hc * kv.vdim + c, v[c] * f);
    }
  } else {
#pragma unroll
    for (int n = 0; n < NB; ++n) {
      const int h = kvh * group + h0 + l16 % gs;
      finish_column<kMaps, VD>(a, o + n * kMaps, m + n * kMaps, l + n * kMaps, row[n], pos[n], live[n] ? h : kvh * group + h0, g);
      if (!live[n]) continue;
      bf16_t* dst = out + (size_t)row[n] * a.out_ld + a.out_col + (size_t)h * kv.vdim;
      const bool vec = (kv.vdim | a.out_ld | a.out_col) % 4 == 0;
#pragma unroll
      for (int i = 0; i < VD; ++i) {
        const int c = i * 16 + g * 4;
        if (i >= vd || c >= kv.vdim) continue;
        const float4_t v = o[n * kMaps][i];
        if (vec) {
          Act<bf16_t>::store4(dst + c, v);
        } else {
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (c + r < kv.vdim) Act<bf16_t>::store(dst + c + r, v[r]);
        }
      }
    }
  }
}

// A slot holds 32 keys: K in planes of 64 elements, 32 rows of 128 bytes, 16-byte chunk c of row r at position c ^ f(r)
// with f = the bits (r>>3 & 3, r>>1 & 1) -- the 16 rows of a fragment, keys 8a + 4b + c, fall on 16 different
// 16-byte slots --; then V as it is cached, per page and value column 32 bytes, halves swapped where bit 3 of the column is
// set, for the same reason.
constexpr int kTileRing = 4;
template <int KD, int VD, int kMaps>
struct TileShape {
  static constexpr int planes = kMaps * KD / 2, k_bytes = planes * 4096, v_groups = VD / 2;  // groups of 32 value columns
  static constexpr int v_bytes = 2 * v_groups * 1024, slot = k_bytes + v_bytes;
  static constexpr int loads = planes + v_groups / 2;  // per wavefront and slot
};

// KD: k_pad / 32 (even), VD: v_pad / 16 (a multiple of 4), NB: column blocks per wavefront.  blockIdx.x: kv head and chunk of its
// query heads -- so that the tiles of a head tend to share an XCD's L2 --, blockIdx.y: tile.
template <int KD, int VD, int NB, int kMaps>
__global__ __launch_bounds__(256, 2) void attn_tile_kernel(nf_window_attention_args a, int gs, int chunks, int tile_tokens, bool all_resident) {
  using S = TileShape<KD, VD, kMaps>;
  constexpr int NC = NB * kMaps;  // sets of columns: a block's maps side by side
  extern __shared__ __attribute__((aligned(1024))) uint8_t ring[];
  const uint32_t lds0 = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) uint8_t*)ring;
  const nf_kv_layout kv = a.kv;
  const int lane = threadIdx.x & 63, l16 = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int group = kv.heads / kv.kv_heads;
  const int kvh = blockIdx.x / chunks, h0 = (blockIdx.x % chunks) * gs;
  const int heads = min(gs, group - h0), tpb = 16 / gs;

  auto tiles_of = [&](int r) { return (a.input_indptr[r + 1] - a.input_indptr[r] + tile_tokens - 1) / tile_tokens; };
  int total = 0;
  for (int r = a.req_begin; r < a.req_begin + a.req_num; ++r) total += tiles_of(r);
  int req = -1, tile = blockIdx.y;
  if (tile >= total) return;
  // Where all workgroups run at once, two to a CU, the second half is dealt out from its end: a CU's two then
  // see about as many keys together as any other's.
  if (all_resident && tile >= total / 2) tile = total - 1 - (tile - total / 2);
  for (int r = a.req_begin; r < a.req_begin + a.req_num; ++r) {
    const int n = tiles_of(r);
    if (tile < n) {
      req = r;
      tile = n - 1 - tile;  // the tiles that see most keys start first
      break;
    }
    tile -= n;
  }
  const int row0 = a.input_indptr[req], len = a.input_indptr[req + 1] - row0;
  const int first_tok = tile * tile_tokens, tok0 = first_tok + wave * NB * tpb;
  const int p0 = a.positions[row0] + first_tok, p1 = p0 + min(tile_tokens, len - first_tok) - 1;  // the workgroup's
  const int w0 = p0 + wave * NB * tpb, w1 = min(w0 + NB * tpb - 1, p1);                          // this wavefront's; none: w0 > w1

  const StepRange steps = visible_steps(a, p0, p1, 32);
  const int all_from = first_seen(a, w1);  // every token of the wavefront sees the keys from here to its own
  const int32_t* pages = a.kv_indices + a.kv_indptr[req];
  const int last_page = p1 / kPage;
  const size_t page_bytes = kv_page_elements(kv) * 2;

  // wavefront w fills key rows 8w .. 8w + 7, and of page w / 2 every second group of 32 value columns
  const int r8 = lane >> 3, vcol = lane >> 1;
  const uint32_t k_off = (uint32_t)((wave & 1) * 8 + r8) * (KD * 64) + (uint32_t)((lane & 7) ^ (wave << 1 | ((r8 >> 1) & 1))) * 16u;
  const uint32_t v_off = (uint32_t)((wave & 1) * 32 + vcol) * 32u + (uint32_t)((lane & 1) ^ ((vcol >> 3) & 1)) * 16u;
  // Page ids of 32 steps at a time, two per step, one per lane: a load of its own in every step would wait for all the steps
  // in flight.
  int ids = 0;
  auto load_step = [&](int it) {
    if (it % 32 == 0) {
      ids = pages[min(steps.at(it + (lane >> 1)) * 2 + (lane & 1), last_page)];
      __builtin_amdgcn_s_waitcnt(0x0F70);
    }
    const int page = __builtin_amdgcn_readlane(ids, it % 32 * 2 + (wave >> 1));
    const uint8_t* base = (const uint8_t*)a.kv_data + (size_t)page * page_bytes;
    const rsrc_t kr = make_rsrc(base + (size_t)kvh * kMaps * kPage * KD * 64, (size_t)kMaps * kPage * KD * 64);
    const rsrc_t vr = make_rsrc(base + ((size_t)kv.kv_heads * kMaps * kPage * KD * 32 + (size_t)kvh * VD * 16 * kPage) * 2, (size_t)VD * 16 * kPage * 2);
    const uint32_t slot = __builtin_amdgcn_readfirstlane(lds0 + (uint32_t)(it % kTileRing) * S::slot);
#pragma unroll
    for (int pl = 0; pl < S::planes; ++pl) load16_to_lds(kr, k_off + pl / (KD / 2) * (kPage * KD * 64) + pl % (KD / 2) * 128, slot + pl * 4096 + wave * 1024);
#pragma unroll
    for (int c = 0; c < S::v_groups; c += 2)
      load16_to_lds(vr, v_off + c * 1024, slot + S::k_bytes + ((wave >> 1) * S::v_groups + (wave & 1) + c) * 1024);
  };
  auto wait_step = [&](int it) {  // this wavefront's loads of step `it`; those of up to two later ones stay in flight
    const int younger = min(steps.total - 1 - it, kTileRing - 2);
    if (younger == 2) __builtin_amdgcn_s_waitcnt(0x0F70 | (2 * S::loads & 15) | ((2 * S::loads >> 4) << 14));
    else if (younger == 1) __builtin_amdgcn_s_waitcnt(0x0F70 | S::loads);
    else __builtin_amdgcn_s_waitcnt(0x0F70);
  };

#pragma unroll 1
  for (int it = 0; it < min(kTileRing - 1, steps.total); ++it) load_step(it);
  int pos[NB], lo_key[NB], row[NB];
  bool live[NB];
  B8 qf[NC][KD];
#pragma unroll
  for (int n = 0; n < NB; ++n) {
    const int tok = tok0 + n * tpb + l16 / gs, hc = l16 % gs;
    live[n] = l16 < tpb * gs && tok < len && hc < heads;
    row[n] = row0 + (live[n] ? tok : first_tok);
    pos[n] = p0 - first_tok + (live[n] ? tok : first_tok);
    lo_key[n] = first_seen(a, pos[n]);
    const bf16_t* q = (const bf16_t*)a.q + ((size_t)row[n] * kv.heads + kvh * group + h0 + (live[n] ? hc : 0)) * (kMaps * KD * 32) + g * 8;
#pragma unroll
    for (int j = 0; j < kMaps * KD; ++j) qf[n * kMaps + j / KD][j % KD].u = *reinterpret_cast<const u32x4*>(q + j * 32);  // columns of no token: never stored
  }
  // Everything has landed once, here: a wait for the queries inside the loop would be one for the steps in flight.
  __builtin_amdgcn_s_waitcnt(0x0F70);

  float4_t o[NC][VD];
  float m[NC], l[NC];
#pragma unroll
  for (int n = 0; n < NC; ++n) {
    m[n] = -1e30f;
    l[n] = 0.f;
#pragma unroll
    for (int i = 0; i < VD; ++i) o[n][i] = float4_t{0.f, 0.f, 0.f, 0.f};
  }
  const ScoreCap cap(a);
  const float scale2 = cap.scale;
  const int key = 8 * (l16 >> 2) + (l16 & 3);  // of score tile 0; tile 1: + 4
  uint32_t kx[2][2];                           // [score tile][chunk half of a plane]
#pragma unroll
  for (int b = 0; b < 2; ++b)
#pragma unroll
    for (int x = 0; x < 2; ++x) {
      const int r = key + 4 * b;
      kx[b][x] = (uint32_t)r * 128u + (uint32_t)((x * 4 + g) ^ (((r >> 3) & 3) << 1 | ((r >> 1) & 1))) * 16u;
    }
  const uint32_t vx = (uint32_t)S::k_bytes + (uint32_t)(g >> 1) * (S::v_groups * 1024) + (uint32_t)l16 * 32u + (uint32_t)((g & 1) ^ (l16 >> 3)) * 16u;

  auto compute = [&](const uint8_t* slot, int base) {
    float4_t s[NC][2];
#pragma unroll
    for (int n = 0; n < NC; ++n)
#pragma unroll
      for (int b = 0; b < 2; ++b) s[n][b] = float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int x = 0; x < kMaps; ++x)
#pragma unroll
      for (int j = 0; j < KD; ++j)
#pragma unroll
        for (int b = 0; b < 2; ++b) {
          B8 k;
          k.u = *reinterpret_cast<const u32x4*>(slot + (x * (KD / 2) + (j >> 1)) * 4096 + kx[b][j & 1]);
#pragma unroll
          for (int n = x; n < NC; n += kMaps) s[n][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k.b, qf[n][j].b, s[n][b], 0, 0, 0);
        }
    if (cap.limit > 0.f)
#pragma unroll
      for (int n = 0; n < NC; ++n)
#pragma unroll
        for (int b = 0; b < 2; ++b) cap.apply(s[n][b]);
    const bool whole = base + 31 <= w0 && (base >= all_from || base + 31 < a.keep_first);
    B8 hi[NC], lo[NC];
#pragma unroll
    for (int n = 0; n < NC; ++n) {
      float mx = -1e30f;
      if (!whole)
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (!sees(pos[n / kMaps], lo_key[n / kMaps], base + 8 * g + 4 * b + r, a.keep_first)) s[n][b][r] = -INFINITY;
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) mx = fmaxf(mx, s[n][b][r]);
      mx = mx > -1e30f ? mx * scale2 : mx;
      // brought to a new maximum only when it has grown by 2^8: weights up to 256 cost nothing in fp32
      if (__any(mx > m[n] + 8.f)) {
        const float m_new = fmaxf(m[n], max_over_lane_groups(mx)), alpha = __builtin_amdgcn_exp2f(m[n] - m_new);
        m[n] = m_new;
        l[n] *= alpha;
#pragma unroll
        for (int i = 0; i < VD; ++i) o[n][i] *= alpha;
      }
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int r = 0; r < 4; r += 2) {
          const float x0 = __builtin_amdgcn_exp2f(fmaf(s[n][b][r], scale2, -m[n])), x1 = __builtin_amdgcn_exp2f(fmaf(s[n][b][r + 1], scale2, -m[n]));
          l[n] += x0 + x1;
          const uint32_t h2 = f32_to_bf16_pair(x0, x1);
          hi[n].w[b * 2 + r / 2] = h2;
          lo[n].w[b * 2 + r / 2] = f32_to_bf16_pair(x0 - __uint_as_float(h2 << 16), x1 - __uint_as_float(h2 & 0xffff0000u));
        }
    }
#pragma unroll
    for (int i = 0; i < VD; ++i) {
      B8 v;
      v.u = *reinterpret_cast<const u32x4*>(slot + vx + i * 512);
#pragma unroll
      for (int n = 0; n < NC; ++n) o[n][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v.b, hi[n].b, o[n][i], 0, 0, 0);
#pragma unroll
      for (int n = 0; n < NC; ++n) o[n][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v.b, lo[n].b, o[n][i], 0, 0, 0);
    }
  };

#pragma unroll 1
  for (int it = 0; it < steps.total; ++it) {
    wait_step(it);
    __syncthreads();  // everyone's part has landed, and everyone is done with the slot of the step before
    if (it + kTileRing - 1 < steps.total) load_step(it + kTileRing - 1);
    const int base = steps.at(it) * 32;
    if (w0 <= w1 && base <= w1) compute(ring + (it % kTileRing) * S::slot, base);
  }

  bf16_t* out = (bf16_t*)a.out;
  const bool vec = (kv.vdim | a.out_ld | a.out_col) % 4 == 0;
#pragma unroll
  for (int n = 0; n < NC; ++n) l[n] = sum_over_lane_groups(l[n]);
#pragma unroll
  for (int n = 0; n < NB; ++n) {
    const int h = kvh * group + h0 + l16 % gs;
    finish_column<kMaps, VD>(a, o + n * kMaps, m + n * kMaps, l + n * kMaps, row[n], pos[n], live[n] ? h : kvh * group + h0, g);
    if (!live[n]) continue;
    bf16_t* dst = out + (size_t)row[n] * a.out_ld + a.out_col + (size_t)h * kv.vdim;
#pragma unroll
    for (int i = 0; i < VD; ++i) {
      const int c = i * 16 + g * 4;
      if (c >= kv.vdim) continue;
      const float4_t v = o[n * kMaps][i];
      if (vec) {
        Act<bf16_t>::store4(dst + c, v);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (c + r < kv.vdim) Act<bf16_t>::store(dst + c + r, v[r]);
      }
    }
  }
}

template <int KD, int VD, int kMaps = 1>
static int launch_tile(const nf_window_attention_args& a, hipStream_t s) {
  constexpr int NB = 2 / kMaps;
  const int group = a.kv.heads / a.kv.kv_heads;
  const int chunks = (group + 15) / 16, gs = (group + chunks - 1) / chunks;
  const int tile_tokens = 4 * NB * (16 / gs);
  const size_t lds = (size_t)kTileRing * TileShape<KD, VD, kMaps>::slot;
  auto kern = attn_tile_kernel<KD, VD, NB, kMaps>;
  static bool attr_set = false;  // benign race: the call is idempotent
  if (!attr_set) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) {
      set_error("nf_window_attention: cannot reserve %zu bytes of LDS: %s", lds, hipGetErrorString(e));
      return NF_ERR_RUNTIME;
    }
    attr_set = true;
  }
  const unsigned tiles = (unsigned)(a.max_rows / tile_tokens + a.req_num);
  kern<<<dim3((unsigned)(a.kv.kv_heads * chunks), tiles), 256, lds, s>>>(a, gs, chunks, tile_tokens, (long long)tiles * a.kv.kv_heads * chunks <= 2 * 256 + 64);
  return check_launch("nf_window_attention (tiles)");
}

template <int KD, int VD, int kMaps = 1>
static int launch_window(const nf_window_attention_args& a, hipStream_t s) {
  const int group = a.kv.heads / a.kv.kv_heads;
  // a kv head's query heads in chunks of at most 16, as equal as possible
  const int chunks = (group + 15) / 16, gs = (group + chunks - 1) / chunks;
  const unsigned gy = (unsigned)(a.kv.kv_heads * chunks);
  if (a.decode) {
    auto lds_of = [&](int w) { return (size_t)w * kMaps * (32 + (size_t)gs * a.kv.v_pad) * sizeof(float); };
    int waves = (long long)a.req_num * gy >= 512 || window_threads(kMaps, VD) < 512 ? 4 : 8;
    while (waves > 1 && lds_of(waves) > 64 * 1024) waves /= 2;
    attn_window_kernel<KD, VD, 1, kMaps, true><<<dim3((unsigned)a.req_num, gy), waves * 64, lds_of(waves), s>>>(a, gs, chunks, 0);
    return check_launch("nf_window_attention (decode)");
  }
  constexpr int NB = KD <= 4 && kMaps == 1 ? 2 : 1;
  const int tile_tokens = 4 * NB * (16 / gs);
  const unsigned tiles = (unsigned)(a.max_rows / tile_tokens + a.req_num);
  attn_window_kernel<KD, VD, NB, kMaps, false><<<dim3(tiles, gy), 256, 0, s>>>(a, gs, chunks, tile_tokens);
  return check_launch("nf_window_attention (prefill)");
}

}  // namespace nf

using namespace nf;

static int check_layout(const char* who, const nf_kv_layout& kv) {
  NF_REQUIRE(kv.dtype == NF_F32 || kv.dtype == NF_BF16, "%s: unknown dtype %d", who, kv.dtype);
  NF_REQUIRE(kv.heads > 0 && kv.kv_heads > 0 && kv.heads % kv.kv_heads == 0, "%s: %d query heads over %d kv heads", who,
             kv.heads, kv.kv_heads);
  NF_REQUIRE(kv.maps == 1 || kv.maps == 2, "%s: %d maps per head", who, kv.maps);
  NF_REQUIRE(kv.page == kPage && kv.dim > 0 && kv.vdim > 0 && kv.dim <= kMaxHeadDim && kv.vdim <= kMaxHeadDim &&
                 kv.k_pad == (kv.dim + 31) / 32 * 32 && kv.v_pad == (kv.vdim + 15) / 16 * 16,
             "%s: page %d, dim %d (pad %d), vdim %d (pad %d): pages of 16, head sizes up to %d", who, kv.page, kv.dim,
             kv.k_pad, kv.vdim, kv.v_pad, kMaxHeadDim);
  return NF_OK;
}

extern "C" {

size_t nf_kv_page_elements(const nf_kv_layout* kv) { return kv ? kv_page_elements(*kv) : 0; }

int nf_qkv_append(const nf_kv_layout* kv, const void* proj, int ld, int q_col, int k_col, int v_col, const float* q_norm,
                  const float* k_norm, float eps, const nf_rotation* rot, const nf_query_temperature* q_temp, const nf_value_form* values,
                  const nf_short_conv* conv, void* q_out, void* kv_data, const int32_t* kv_indptr, const int32_t* kv_indices, const int32_t* rev_input_indptr,
                  const int32_t* positions, int rows, nf_stream_t stream) {
  const char* who = "nf_qkv_append";
  NF_REQUIRE(kv && rot, "%s: null pointer", who);
  int rc = check_layout(who, *kv);
  if (rc) return rc;
  NF_REQUIRE(rot->dims >= 0 && rot->dims % 2 == 0 && rot->dims <= kv->dim && (rot->dims == 0 || rot->table),
             "%s: %d of %d dimensions rotated", who, rot->dims, kv->dim);
  NF_REQUIRE(rows >= 0 && q_col >= 0 && k_col >= 0 && v_col >= 0 && q_col + kv->heads * kv->maps * kv->dim <= ld &&
                 k_col + kv->kv_heads * kv->maps * kv->dim <= ld && v_col + kv->kv_heads * kv->vdim <= ld,
             "%s: columns %d %d %d do not fit rows of %d", who, q_col, k_col, v_col, ld);
  NF_REQUIRE(!q_temp || q_temp->every > 0, "%s: a query temperature with blocks of %d positions", who, q_temp ? q_temp->every : 0);
  const nf_short_conv cv = conv ? *conv : nf_short_conv{};
  NF_REQUIRE(!conv || (cv.taps >= 1 && cv.taps <= 64 && cv.weight && cv.input_indptr && (cv.taps == 1 || (cv.state && cv.state_slots))),
             "%s: a convolution of %d taps (1..64) needs weights, a state and slots", who, cv.taps);
  const nf_value_form vf = values ? *values : nf_value_form{};
  NF_REQUIRE(vf.rot.dims >= 0 && vf.rot.dims % 2 == 0 && vf.rot.dims <= kv->vdim && (vf.rot.dims == 0 || (vf.rot.table && vf.rot.interleaved)),
             "%s: %d of %d value columns rotated, in pairs side by side", who, vf.rot.dims, kv->vdim);
  const nf_query_temperature temp = q_temp ? *q_temp : nf_query_temperature{0.f, 0};
  if (rows == 0) return NF_OK;
  NF_REQUIRE(proj && q_out && kv_data && kv_indptr && kv_indices && rev_input_indptr && positions, "%s: null pointer", who);
  hipStream_t s = (hipStream_t)stream;
  const size_t four = 4 * (kv->dtype == NF_BF16 ? 2 : 4);
  const uintptr_t places = (uintptr_t)proj | (uintptr_t)cv.weight | (uintptr_t)cv.state | (uintptr_t)q_out | (uintptr_t)kv_data;
  const int sizes = kv->dim | kv->vdim | ld | q_col | k_col | v_col, turned = rot->interleaved ? rot->dims : rot->dims / 2;
  if (sizes % 4 == 0 && places % four == 0 && (turned | vf.rot.dims) % 4 == 0 && rows < (1 << 20)) {
    const bool few = rows < 1024;
    auto go = [&](auto type, auto vec, auto run) {
      using T = decltype(type);
      constexpr int kRun = decltype(run)::value;
      const int value_blocks = few ? 0 : (rows + 15) / 16 * kv->kv_heads;
      const int jobs = (kv->heads + kv->kv_heads) * kv->maps + (few ? kv->kv_heads : 0);
      const int blocks = value_blocks + (rows + kRun - 1) / kRun * ((jobs + 15) / 16);
      auto launch = [&](auto kern) {
        kern<<<(unsigned)blocks, 256, 0, s>>>(*kv, (const T*)proj, ld, q_col, k_col, v_col, q_norm, k_norm, eps, *rot, temp, vf, cv, (T*)q_out,
                                              (T*)kv_data, kv_indptr, kv_indices, rev_input_indptr, positions, rows, value_blocks);
        return check_launch(who);
      };
      return cv.taps > 0 ? launch(qkv_append4_kernel<T, decltype(vec)::value, kRun, true>) : launch(qkv_append4_kernel<T, decltype(vec)::value, kRun, false>);
    };
    auto sized = [&](auto type, auto run) {
      const int widest = few ? std::max(kv->k_pad, kv->v_pad) : kv->k_pad;
      return widest <= 64 ? go(type, Int<1>{}, run) : widest <= 128 ? go(type, Int<2>{}, run) : go(type, Int<4>{}, run);
    };
    if (kv->dtype == NF_F32) return sized(float{}, Int<1>{});
    return few ? sized(bf16_t{}, Int<1>{}) : sized(bf16_t{}, Int<2>{});
  }
  const dim3 grid((unsigned)rows, (unsigned)(((kv->heads + kv->kv_heads) * kv->maps + kv->kv_heads + 3) / 4));
  if (kv->dtype == NF_BF16)
    qkv_append_kernel<bf16_t><<<grid, 256, 0, s>>>(*kv, (const bf16_t*)proj, ld, q_col, k_col, v_col, q_norm, k_norm, eps, *rot, temp, vf, cv,
                                                   (bf16_t*)q_out, (bf16_t*)kv_data, kv_indptr, kv_indices, rev_input_indptr,
                                                   positions);
  else
    qkv_append_kernel<float><<<grid, 256, 0, s>>>(*kv, (const float*)proj, ld, q_col, k_col, v_col, q_norm, k_norm, eps, *rot, temp, vf, cv,
                                                  (float*)q_out, (float*)kv_data, kv_indptr, kv_indices, rev_input_indptr,
                                                  positions);
  return check_launch(who);
}

int nf_conv_state(int dtype, const void* proj, int ld, const nf_short_conv* conv, const int32_t* positions, int req_begin, int req_num,
                  nf_stream_t stream) {
  const char* who = "nf_conv_state";
  NF_REQUIRE(dtype == NF_F32 || dtype == NF_BF16, "%s: unknown dtype %d", who, dtype);
  NF_REQUIRE(conv && conv->taps >= 1 && conv->taps <= 64 && ld > 0 && ld % 8 == 0 && req_begin >= 0 && req_num >= 0, "%s: taps or rows", who);
  if (req_num == 0 || conv->taps == 1) return NF_OK;
  NF_REQUIRE(proj && positions && conv->state && conv->input_indptr && conv->state_slots, "%s: null pointer", who);
  NF_REQUIRE(((uintptr_t)proj | (uintptr_t)conv->state) % 16 == 0, "%s: operands must be 16-byte aligned", who);
  const int per = 256 * (dtype == NF_BF16 ? 8 : 4);
  const dim3 grid((unsigned)req_num, (unsigned)((ld + per - 1) / per));
  if (dtype == NF_BF16) conv_state_kernel<bf16_t><<<grid, 256, 0, (hipStream_t)stream>>>((const bf16_t*)proj, ld, *conv, positions, req_begin);
  else conv_state_kernel<float><<<grid, 256, 0, (hipStream_t)stream>>>((const float*)proj, ld, *conv, positions, req_begin);
  return check_launch(who);
}

int nf_window_attention(const nf_window_attention_args* args, nf_stream_t stream) {
  const char* who = "nf_window_attention";
  NF_REQUIRE(args, "%s: null pointer", who);
  const nf_window_attention_args& a = *args;
  int rc = check_layout(who, a.kv);
  if (rc) return rc;
  NF_REQUIRE(a.req_num >= 0 && a.req_begin >= 0 && a.max_rows >= 0 && a.row_begin >= 0 && a.keep_first >= 0,
             "%s: requests %d + %d, rows %d + %d, keep_first %d", who, a.req_begin, a.req_num, a.row_begin, a.max_rows,
             a.keep_first);
  NF_REQUIRE(a.out_col >= 0 && a.out_col + a.kv.heads * a.kv.vdim <= a.out_ld, "%s: output columns %d + %d of %d", who,
             a.out_col, a.kv.heads * a.kv.vdim, a.out_ld);
  NF_REQUIRE(!a.gate || a.gate_ld >= a.kv.heads, "%s: gate rows of %d for %d heads", who, a.gate_ld, a.kv.heads);
  NF_REQUIRE(a.kv.maps == 1 || !a.sink, "%s: a sink with two maps", who);
  NF_REQUIRE(a.out_rot.dims == 0 || (a.out_rot.dims == a.kv.vdim && a.kv.vdim % 2 == 0 && a.out_rot.table && a.out_rot.interleaved),
             "%s: %d of %d output columns turned back, in pairs side by side", who, a.out_rot.dims, a.kv.vdim);
  NF_REQUIRE(a.chunk >= 0, "%s: chunks of %d", who, a.chunk);
  NF_REQUIRE(a.softcap >= 0.f && (!a.head_norm || a.head_eps >= 0.f), "%s: cap %g, eps %g", who, a.softcap, a.head_eps);
  NF_REQUIRE(!a.decode || a.max_rows == a.req_num, "%s: %d decode requests with %d rows", who, a.req_num, a.max_rows);
  if (a.req_num == 0 || a.max_rows == 0) return NF_OK;
  NF_REQUIRE(a.q && a.out && a.kv_data && a.input_indptr && a.kv_indptr && a.kv_indices && a.rev_input_indptr && a.positions,
             "%s: null pointer", who);
  hipStream_t s = (hipStream_t)stream;
  NF_REQUIRE(a.kv.heads <= 65535, "%s: %d heads exceed the grid", who, a.kv.heads);
  if (a.kv.dtype == NF_F32) {
    attn_rows_kernel<float><<<dim3((unsigned)a.max_rows, (unsigned)a.kv.heads), 64, 0, s>>>(a);
    return check_launch(who);
  }
  const int kd = a.kv.k_pad / 32, vd = a.kv.v_pad / 16;
  // the matrix kernel takes the maximum before it scales; keys of two maps beyond 128 columns do not fit its registers
  if (!(a.scale > 0.f) || (a.kv.maps == 2 && kd > 4)) {
    attn_rows_kernel<bf16_t><<<dim3((unsigned)a.max_rows, (unsigned)a.kv.heads), 64, 0, s>>>(a);
    return check_launch(who);
  }
  const bool tiles = !a.decode && (long long)a.max_rows + a.req_num <= 65535;
  if (a.kv.maps == 2) {
    if (tiles && kd == 2 && vd == 4) return launch_tile<2, 4, 2>(a, s);
    if (tiles && kd == 2 && vd == 8) return launch_tile<2, 8, 2>(a, s);
    if (tiles && kd == 4 && vd == 8) return launch_tile<4, 8, 2>(a, s);
    if (tiles && kd == 4 && vd == 16) return launch_tile<4, 16, 2>(a, s);
    if (kd <= 2 && vd <= 8) return launch_window<2, 8, 2>(a, s);
    return launch_window<4, 16, 2>(a, s);
  }
  if (tiles) {
    if (kd == 2 && vd == 4) return launch_tile<2, 4>(a, s);
    if (kd == 4 && vd == 8) return launch_tile<4, 8>(a, s);
    if (kd == 6 && vd == 8) return launch_tile<6, 8>(a, s);
  }
  if (kd <= 2 && vd <= 4) return launch_window<2, 4>(a, s);
  if (kd <= 4 && vd <= 8) return launch_window<4, 8>(a, s);
  return launch_window<8, 16>(a, s);
}

}  // extern "C"
