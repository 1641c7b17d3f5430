// Linear recurrences of the layer-stack pipeline: a state S [dim][vdim] per head, fp32.  A token scales
// the state's rows, adds the outer product of its key and value, and reads the state with its query:
// after the update (FIXED_DECAY), or before it with the token's own key weighted by u (TOKEN_DECAY).
// With S the state before the token, both reads are
//     o = c (q . S) + b v,     b = q . k  or  q . (u * k),     c = the decay  or  1.
// Everything between the loaded projections and the stored output is fp32: rotation, decays,
// products, state, the per-head norm and the gate.
//
// recur_seq_kernel: one workgroup per (request, head) holds the head's state in registers and walks
// the request's rows, a few at a time through LDS.  Decode (one row): the state is streamed in, used,
// and streamed out once.
#include <algorithm>
#include <cmath>

#include "layer_common.h"

namespace nf {

constexpr int kMaxStateDim = 256;

struct RecurrenceDims {
  int kp, vp;  // dim and vdim padded to 16
};
__host__ __device__ inline RecurrenceDims padded(int dim, int vdim) { return {(dim + 15) / 16 * 16, (vdim + 15) / 16 * 16}; }

// Element d of a row's head vector `src`, rotated to position `pos`.
template <class T>
__device__ __forceinline__ float load_rotated(const T* src, int d, const nf_rotation& rot, int pos) {
  const float y = Act<T>::load(src + d);
  const int half = rot.dims / 2;
  if (d >= 2 * half) return y;
  const int f = rot.interleaved ? d >> 1 : (d < half ? d : d - half);
  const bool first = rot.interleaved ? !(d & 1) : d < half;
  const float other = Act<T>::load(src + (rot.interleaved ? d ^ 1 : (first ? d + half : d - half)));
  const float cs = rot.table[((size_t)pos * half + f) * 2], sn = rot.table[((size_t)pos * half + f) * 2 + 1];
  return first ? y * cs - other * sn : y * cs + other * sn;
}

// log2 of the factor that key channel `col` (over all heads) is multiplied by at a row.  Limited to
// 2^-126: a smaller factor leaves nothing of a state in fp32, and sums of logs stay finite.
__device__ __forceinline__ float token_log2_decay(const nf_recurrence_args& a, int row, int col) {
  float z = a.w0[col];
  for (int s = 0; s < a.z_shares; ++s) z += a.z[((size_t)s * a.total_rows + row) * a.z_ld + col];
  return fmaxf(-expf(z) * 1.44269504088896340736f, -126.f);
}

template <class T, int NP, int KIND>
__global__ __launch_bounds__(1024) void recur_seq_kernel(nf_recurrence_args a, int tb) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const RecurrenceDims pd = padded(a.dim, a.vdim);
  const int req = a.req_begin + blockIdx.x, h = blockIdx.y;
  const int ns = blockDim.x / 256, vw = ns * 64;
  float* sq = lds;                   // [tb][kp]
  float* sk = sq + tb * pd.kp;       // [tb][kp]
  float* sw = sk + tb * pd.kp;       // [tb][kp] (TOKEN_DECAY)
  float* sv = sw + (KIND == NF_RECURRENCE_TOKEN_DECAY ? tb * pd.kp : 0);  // [tb][vw]
  float* sp = sv + tb * vw;          // [tb][4][vw]
  float* sb = sp + tb * 4 * vw;      // [tb]

  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, n_waves = blockDim.x >> 6;
  const int slice = tid >> 8, col = slice * 64 + (tid & 15) * 4, krow = (tid & 255) >> 4, swave = (tid & 255) >> 6;
  const int row0 = a.input_indptr[req], row1 = a.input_indptr[req + 1];
  if (row0 >= row1) return;
  const int slot = a.state_slots[req];
  float* state = a.state + ((size_t)slot * a.heads + h) * pd.kp * pd.vp;
  const bool fresh = a.positions[row0] == 0;
  const float decay = KIND == NF_RECURRENCE_FIXED_DECAY ? exp2f(a.log2_decay[h]) : 1.f;

  float4_t S[NP];
#pragma unroll
  for (int i = 0; i < NP; ++i) {
    const int k = krow + 16 * i;
    S[i] = float4_t{0.f, 0.f, 0.f, 0.f};
    if (!fresh && k < pd.kp && col < pd.vp) S[i] = *reinterpret_cast<const float4_t*>(state + (size_t)k * pd.vp + col);
  }

  for (int r0 = row0; r0 < row1; r0 += tb) {
    const int n = min(tb, row1 - r0);
    for (int e = tid; e < n * pd.kp; e += blockDim.x) {
      const int t = e / pd.kp, d = e % pd.kp, row = r0 + t;
      float q = 0.f, k = 0.f, w = 1.f;
      if (d < a.dim) {
        const T* qp = (const T*)a.q + (size_t)row * a.q_ld + (size_t)h * a.dim;
        const T* kp = (const T*)a.k + (size_t)row * a.k_ld + (size_t)h * a.dim;
        if constexpr (KIND == NF_RECURRENCE_FIXED_DECAY) {
          const int pos = a.positions[row];
          q = load_rotated(qp, d, a.rot, pos);
          k = load_rotated(kp, d, a.rot, pos) * a.k_scale;
        } else {
          q = Act<T>::load(qp + d);
          k = Act<T>::load(kp + d);
          w = exp2f(token_log2_decay(a, row, h * a.dim + d));
        }
      }
      sq[e] = q;
      sk[e] = k;
      if constexpr (KIND == NF_RECURRENCE_TOKEN_DECAY) sw[e] = w;
    }
    for (int e = tid; e < n * vw; e += blockDim.x) {
      const int t = e / vw, c = e % vw;
      sv[e] = c < a.vdim ? Act<T>::load((const T*)a.v + (size_t)(r0 + t) * a.v_ld + (size_t)h * a.vdim + c) : 0.f;
    }
    __syncthreads();
    for (int t = wave; t < n; t += n_waves) {
      float b = 0.f;
      for (int d = lane; d < a.dim; d += 64)
        b += sq[t * pd.kp + d] * sk[t * pd.kp + d] * (KIND == NF_RECURRENCE_TOKEN_DECAY ? a.u[(size_t)h * a.dim + d] : 1.f);
      b = wave_sum(b);
      if (lane == 0) sb[t] = b;
    }
    for (int t = 0; t < n; ++t) {
      const float4_t v = *reinterpret_cast<const float4_t*>(sv + t * vw + col);
      float4_t o{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < NP; ++i) {
        const int k = min(krow + 16 * i, pd.kp - 1);  // rows past the state's last hold zeros of no effect
        const float w = KIND == NF_RECURRENCE_TOKEN_DECAY ? sw[t * pd.kp + k] : decay;
        o += S[i] * sq[t * pd.kp + k];
        S[i] = S[i] * w + v * sk[t * pd.kp + k];
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        o[e] += __shfl_xor(o[e], 16, 64);
        o[e] += __shfl_xor(o[e], 32, 64);
      }
      if (lane < 16) *reinterpret_cast<float4_t*>(sp + (t * 4 + swave) * vw + col) = o;
    }
    __syncthreads();
    // per row: the four partial sums, the current token's own term, norm, gate
    for (int t = wave; t < n; t += n_waves) {
      const int row = r0 + t;
      float o[kMaxStateDim / 64], sqs = 0.f;
#pragma unroll
      for (int e = 0; e < kMaxStateDim / 64; ++e) {
        const int c = e * 64 + lane;
        o[e] = 0.f;
        if (c < a.vdim) {
          const float* p = sp + (size_t)t * 4 * vw + c;
          o[e] = (p[0] + p[vw] + p[2 * vw] + p[3 * vw]) * decay + sb[t] * sv[t * vw + c];
        }
        sqs += o[e] * o[e];
      }
      const float inv = a.out_scale / sqrtf(wave_sum(sqs) / (float)a.vdim + a.eps);
#pragma unroll
      for (int e = 0; e < kMaxStateDim / 64; ++e) {
        const int c = e * 64 + lane;
        if (c >= a.vdim) continue;
        const int hc = h * a.vdim + c;
        float y = o[e] * inv * silu_f32(Act<T>::load((const T*)a.g + (size_t)row * a.g_ld + hc));
        if (a.norm_weight) y *= a.norm_weight[hc];
        Act<T>::store((T*)a.out + (size_t)row * a.out_ld + a.out_col + hc, y);
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < NP; ++i) {
    const int k = krow + 16 * i;
    if (k < pd.kp && col < pd.vp) *reinterpret_cast<float4_t*>(state + (size_t)k * pd.vp + col) = S[i];
  }
  if (a.shift_x && h == 0)
    for (int c = tid * 4; c < a.shift_ld; c += blockDim.x * 4)
      *reinterpret_cast<float4_t*>(a.shift_state + (size_t)slot * a.shift_ld + c) =
          *reinterpret_cast<const float4_t*>(a.shift_x + (size_t)(row1 - 1) * a.shift_ld + c);
}

template <class T, int KIND>
static int launch_seq(const nf_recurrence_args& a, hipStream_t s) {
  const RecurrenceDims pd = padded(a.dim, a.vdim);
  const int ns = (pd.vp + 63) / 64, vw = ns * 64;
  // decode: one row per request; else as many rows at a time as 64 KB of LDS hold, at most 8
  auto lds_of = [&](int tb) {
    return ((size_t)tb * pd.kp * (KIND == NF_RECURRENCE_TOKEN_DECAY ? 3 : 2) + (size_t)tb * vw * 5 + tb) * sizeof(float);
  };
  int tb = a.rows == a.req_num ? 1 : 8;
  while (tb > 1 && lds_of(tb) > 64 * 1024) tb /= 2;
  const dim3 grid((unsigned)a.req_num, (unsigned)a.heads);
  auto go = [&](auto np) {
    recur_seq_kernel<T, decltype(np)::value, KIND><<<grid, ns * 256, lds_of(tb), s>>>(a, tb);
    return check_launch("nf_linear_recurrence");
  };
  const int np = pd.kp / 16;
  if (np <= 2) return go(ic<2>{});
  if (np <= 4) return go(ic<4>{});
  if (np <= 8) return go(ic<8>{});
  return go(ic<16>{});
}

}  // namespace nf

using namespace nf;

extern "C" {

size_t nf_recurrence_state_elements(int dim, int vdim) {
  if (dim <= 0 || vdim <= 0) return 0;
  const RecurrenceDims pd = padded(dim, vdim);
  return (size_t)pd.kp * pd.vp;
}

size_t nf_recurrence_workspace_bytes(int heads, int dim, int vdim, int max_rows, int max_requests) { return 0; }

int nf_linear_recurrence(const nf_recurrence_args* args, nf_stream_t stream) {
  const char* who = "nf_linear_recurrence";
  NF_REQUIRE(args, "%s: null pointer", who);
  const nf_recurrence_args& a = *args;
  NF_REQUIRE(a.dtype == NF_F32 || a.dtype == NF_BF16, "%s: unknown dtype %d", who, a.dtype);
  NF_REQUIRE(a.kind == NF_RECURRENCE_FIXED_DECAY || a.kind == NF_RECURRENCE_TOKEN_DECAY, "%s: unknown kind %d", who, a.kind);
  NF_REQUIRE(a.heads > 0 && a.heads <= 65535 && a.dim > 0 && a.vdim > 0 && a.dim <= kMaxStateDim && a.vdim <= kMaxStateDim,
             "%s: %d heads of %d x %d (at most %d)", who, a.heads, a.dim, a.vdim, kMaxStateDim);
  NF_REQUIRE(a.req_num >= 0 && a.req_begin >= 0 && a.rows >= a.req_num && a.row_begin >= 0, "%s: %d requests with %d rows",
             who, a.req_num, a.rows);
  NF_REQUIRE(a.q_ld >= a.heads * a.dim && a.k_ld >= a.heads * a.dim && a.v_ld >= a.heads * a.vdim && a.g_ld >= a.heads * a.vdim &&
                 a.out_col >= 0 && a.out_col + a.heads * a.vdim <= a.out_ld,
             "%s: row strides too small", who);
  if (a.req_num == 0) return NF_OK;
  NF_REQUIRE(a.q && a.k && a.v && a.g && a.state && a.out && a.input_indptr && a.positions && a.state_slots,
             "%s: null pointer", who);
  if (a.kind == NF_RECURRENCE_FIXED_DECAY) {
    NF_REQUIRE(a.log2_decay && a.rot.dims >= 0 && a.rot.dims % 2 == 0 && a.rot.dims <= a.dim && (a.rot.dims == 0 || a.rot.table),
               "%s: decay or rotation missing", who);
  } else {
    NF_REQUIRE(a.z && a.w0 && a.u && a.z_shares >= 1 && a.z_shares <= kMaxShares && a.z_ld >= a.heads * a.dim &&
                   a.total_rows >= a.row_begin + a.rows,
               "%s: token decay inputs missing", who);
  }
  NF_REQUIRE(!a.shift_x || (a.shift_state && a.shift_ld > 0 && a.shift_ld % 4 == 0), "%s: shift state missing", who);
  hipStream_t s = (hipStream_t)stream;
  if (a.dtype == NF_BF16)
    return a.kind == NF_RECURRENCE_FIXED_DECAY ? launch_seq<bf16_t, NF_RECURRENCE_FIXED_DECAY>(a, s)
                                               : launch_seq<bf16_t, NF_RECURRENCE_TOKEN_DECAY>(a, s);
  return a.kind == NF_RECURRENCE_FIXED_DECAY ? launch_seq<float, NF_RECURRENCE_FIXED_DECAY>(a, s)
                                             : launch_seq<float, NF_RECURRENCE_TOKEN_DECAY>(a, s);
}

}  // extern "C"
