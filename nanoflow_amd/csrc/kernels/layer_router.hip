// Routing of a mixture of experts: scores, choice, and the order of the chosen rows by expert.
//
// route_rows_kernel: one wavefront per token, its scores in registers (fp32 softmax over all outputs, or a sigmoid of each), groups of
//   outputs closed by the rank of their largest entry, the `top` largest taken one after the other, then the
//   experts that every token has.
// route_plan_kernel: one workgroup counts the rows of every expert, places them (an expert's rows consecutive)
//   and lists the m tiles of the grouped product.  The place of a row inside its expert's run
//   depends on the order of LDS atomics; nothing computed from it does.
#include <algorithm>
#include <cmath>

#include "layer_common.h"

namespace nf {

constexpr int kMaxOutputs = 1024, kMaxTop = 64;

template <int kPer>  // outputs per lane
__global__ __launch_bounds__(256) void route_rows_kernel(nf_route_args a, int32_t* __restrict__ choice, float* __restrict__ weight) {
  __shared__ float entry[4][kPer * 64], best_of[4][kPer * 64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, t = blockIdx.x * 4 + wave;
  const bool live = t < a.rows;
  const float* __restrict__ z = a.z + (size_t)(live ? t : 0) * a.ld;
  const int shares = a.shares, outputs = a.outputs, per_token = a.top + a.always;
  const size_t slice = (size_t)a.rows * a.ld;
  float s[kPer], c[kPer];
  float mx = -INFINITY;
#pragma unroll
  for (int i = 0; i < kPer; ++i) {
    const int o = i * 64 + lane;
    s[i] = -INFINITY;
    if (o < outputs) {
      float part[kMaxShares];  // in flight together
#pragma unroll
      for (int p = 0; p < kMaxShares; ++p) part[p] = p < shares ? z[p * slice + o] : 0.f;
      s[i] = part[0];
#pragma unroll
      for (int p = 1; p < kMaxShares; ++p) s[i] += part[p];
    }
    mx = fmaxf(mx, s[i]);
  }
#pragma unroll
  for (int m = 32; m > 0; m >>= 1) mx = fmaxf(mx, __shfl_xor(mx, m, 64));
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < kPer; ++i) {
    const bool is = i * 64 + lane < outputs;
    if (a.scores == NF_SCORES_SIGMOID) s[i] = is ? 1.f / (1.f + expf(-s[i])) : 0.f;
    else s[i] = is ? expf(s[i] - mx) : 0.f;
    sum += s[i];
  }
  sum = a.scores == NF_SCORES_SIGMOID ? 1.f : wave_sum(sum);
#pragma unroll
  for (int i = 0; i < kPer; ++i) {
    const int o = i * 64 + lane;
    s[i] /= sum;
    c[i] = o < outputs ? s[i] + (a.correction ? a.correction[o] : 0.f) : -INFINITY;
  }
  if (a.groups > 1) {  // the same for every wavefront: the barriers are met by all
    const int size = outputs / a.groups;
#pragma unroll
    for (int i = 0; i < kPer; ++i) entry[wave][i * 64 + lane] = c[i];
    __syncthreads();
    for (int g = lane; g < a.groups; g += 64) {
      float b = entry[wave][g * size];
      for (int e = 1; e < size; ++e) b = fmaxf(b, entry[wave][g * size + e]);
      best_of[wave][g] = b;
    }
    __syncthreads();
    for (int g = lane; g < a.groups; g += 64) {
      const float b = best_of[wave][g];
      int ahead = 0;  // groups with a larger entry, or as large and before it
      for (int o = 0; o < a.groups; ++o) ahead += best_of[wave][o] > b || (best_of[wave][o] == b && o < g);
      entry[wave][g] = ahead < a.keep_groups ? 1.f : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < kPer; ++i) {
      const int o = i * 64 + lane;
      if (o < outputs && entry[wave][o / size] == 0.f) c[i] = -INFINITY;
    }
  }
  if (!live) return;
  for (int k = 0; k < a.top; ++k) {
    float best = -INFINITY, w = 0.f;
    int at = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < kPer; ++i)
      if (c[i] > best) {  // the smallest of equal ones: i ascends
        best = c[i];
        at = i * 64 + lane;
        w = s[i];
      }
#pragma unroll
    for (int m = 32; m > 0; m >>= 1) {
      const float b2 = __shfl_xor(best, m, 64), w2 = __shfl_xor(w, m, 64);
      const int a2 = __shfl_xor(at, m, 64);
      if (b2 > best || (b2 == best && a2 < at)) {
        best = b2;
        at = a2;
        w = w2;
      }
    }
    if (at >= outputs) at = 0, w = 0.f;  // scores that are no numbers: a valid index all the same
#pragma unroll
    for (int i = 0; i < kPer; ++i)
      if (i * 64 + lane == at) c[i] = -INFINITY;
    if (lane == 0) {
      choice[(size_t)t * per_token + k] = at;
      weight[(size_t)t * per_token + k] = w * a.scale;
    }
  }
  if (lane < a.always) {
    float g = 0.f;
    if (!a.always_plain)
      for (int p = 0; p < shares; ++p) g += z[p * slice + outputs];
    choice[(size_t)t * per_token + a.top + lane] = outputs + lane;
    weight[(size_t)t * per_token + a.top + lane] = a.always_plain ? 1.f : 1.f / (1.f + expf(-g));
  }
}

// experts: of the grouped product, the last `always` of which have every token's row, in the tokens' order.
__global__ __launch_bounds__(1024) void route_plan_kernel(nf_routing r, int rows, int top, int always, int experts) {
  __shared__ int count[kMaxOutputs], first[kMaxOutputs], tile0[kMaxOutputs], wave_rows[16], wave_tiles[16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, routed = experts - always, per_token = top + always, n = rows * per_token;
  count[tid] = tid >= routed && tid < experts ? rows : 0;
  __syncthreads();
  constexpr int kAhead = 4;  // choices of a thread requested at once
  for (int i0 = tid; i0 < n; i0 += kAhead * 1024) {
    int e[kAhead];
#pragma unroll
    for (int k = 0; k < kAhead; ++k) e[k] = r.choice[min(i0 + k * 1024, n - 1)];
#pragma unroll
    for (int k = 0; k < kAhead; ++k) {
      const int i = i0 + k * 1024;
      if (i < n && i % per_token < top && e[k] < routed) atomicAdd(&count[e[k]], 1);
    }
  }
  __syncthreads();
  // exclusive sums over the experts: rows, tiles
  const int c = count[tid], tiles = (c + r.tile_rows - 1) / r.tile_rows;
  int rows_to = c, tiles_to = tiles;
#pragma unroll
  for (int d = 1; d < 64; d <<= 1) {
    const int a = __shfl_up(rows_to, d, 64), b = __shfl_up(tiles_to, d, 64);
    if (lane >= d) {
      rows_to += a;
      tiles_to += b;
    }
  }
  if (lane == 63) {
    wave_rows[wave] = rows_to;
    wave_tiles[wave] = tiles_to;
  }
  __syncthreads();
  for (int w = 0; w < wave; ++w) {
    rows_to += wave_rows[w];
    tiles_to += wave_tiles[w];
  }
  first[tid] = rows_to - c;
  tile0[tid] = tiles_to - tiles;
  if (tid < experts) {
    r.offsets[tid + 1] = rows_to;
    if (tid == 0) r.offsets[0] = 0;
    if (tid == experts - 1) *r.n_tiles = tiles_to;
    for (int i = 0; i < tiles; ++i) {
      r.tile_group[tile0[tid] + i] = tid;
      r.tile_row[tile0[tid] + i] = i * r.tile_rows;
    }
  }
  __syncthreads();
  for (int i0 = tid; i0 < n; i0 += kAhead * 1024) {
    int choice[kAhead];
    float weight[kAhead];
#pragma unroll
    for (int x = 0; x < kAhead; ++x) {
      choice[x] = r.choice[min(i0 + x * 1024, n - 1)];
      weight[x] = r.weight[min(i0 + x * 1024, n - 1)];
    }
#pragma unroll
    for (int x = 0; x < kAhead; ++x) {
      const int i = i0 + x * 1024, t = i / per_token, k = i % per_token, e = choice[x];
      if (i >= n) break;
      int at = -1;
      if (k >= top) at = first[routed + k - top] + t;
      else if (e < routed) at = atomicAdd(&first[e], 1);
      if (at >= 0) {
        r.row_of[at] = t;
        if (r.row_weight) r.row_weight[at] = weight[x];
      }
      r.place[i] = at;
    }
  }
}

}  // namespace nf

using namespace nf;

extern "C" {

int nf_routing_max_tiles(int sorted_rows, int experts, int tile_rows) {
  return sorted_rows > 0 && tile_rows > 0 ? sorted_rows / tile_rows + std::min(experts, sorted_rows) : 0;
}

int nf_route(const nf_route_args* args, const nf_routing* routing, nf_stream_t stream) {
  const char* who = "nf_route";
  NF_REQUIRE(args && routing, "%s: null pointer", who);
  const nf_route_args& a = *args;
  NF_REQUIRE(a.outputs > 0 && a.outputs <= kMaxOutputs && a.experts > 0 && a.experts <= a.outputs && a.top > 0 && a.always >= 0 &&
                 a.top <= a.outputs && a.top + a.always <= kMaxTop && a.experts + a.always <= kMaxOutputs,
             "%s: top %d and %d more of %d outputs, %d experts (at most %d outputs, %d per token)", who, a.top, a.always, a.outputs, a.experts,
             kMaxOutputs, kMaxTop);
  NF_REQUIRE(a.groups <= 1 || (a.outputs % a.groups == 0 && a.keep_groups > 0 && a.keep_groups <= a.groups &&
                               a.top <= a.outputs / a.groups * a.keep_groups),
             "%s: top %d of the outputs of %d of %d groups of %d", who, a.top, a.keep_groups, a.groups, a.outputs);
  const int per_token = a.top + a.always;
  NF_REQUIRE(a.rows >= 0 && (long long)a.rows * per_token < (1ll << 31) && a.ld >= a.outputs + (a.always > 0 && !a.always_plain) && a.shares >= 1 &&
                 a.shares <= kMaxShares && routing->tile_rows > 0,
             "%s: rows=%d ld=%d shares=%d tile_rows=%d", who, a.rows, a.ld, a.shares, routing->tile_rows);
  NF_REQUIRE(a.scores == NF_SCORES_SOFTMAX || a.scores == NF_SCORES_SIGMOID, "%s: unknown scores %d", who, a.scores);
  if (a.rows == 0) return NF_OK;
  const nf_routing& r = *routing;
  NF_REQUIRE(a.z && r.choice && r.weight && r.place && r.row_of && r.offsets && r.tile_group && r.tile_row && r.n_tiles, "%s: null pointer", who);
  hipStream_t s = (hipStream_t)stream;
  auto go = [&](auto per) {
    route_rows_kernel<decltype(per)::value><<<(a.rows + 3) / 4, 256, 0, s>>>(a, r.choice, r.weight);
    return check_launch(who);
  };
  const int per = (a.outputs + 63) / 64;
  const int rc = per <= 1 ? go(ic<1>{}) : per <= 2 ? go(ic<2>{}) : per <= 4 ? go(ic<4>{}) : per <= 8 ? go(ic<8>{}) : go(ic<16>{});
  if (rc) return rc;
  route_plan_kernel<<<1, 1024, 0, s>>>(r, a.rows, a.top, a.always, a.experts + a.always);
  return check_launch("nf_route (plan)");
}

}  // extern "C"
