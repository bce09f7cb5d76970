// What a mixer with a token shift and data-dependent decays reads, and the rows of a looped pass:
//
//   token_shift_kernel     out[t, s, :] = h[t] + (h[t - 1] - h[t]) * mu[s, :]   for every stream s of a mixer's input
//   low_rank_decay_kernel  a[t, c] = exp(-exp(sum_r w[r, c] tanh(p[t, r]) + w0[c]))
//   concat_rows_kernel     out[t] = [x[t] | y[t]]
//
// A request's tokens of this step are rows first .. first + count - 1 (seq_meta [S, 4]: state slot, first row, count,
// position of the first).  The row before a request's first one of the step is the slot's tail (zeros at the start).
// Differences, sums, tanh and exponentials are 32-bit whatever the element types are.
#include "api.h"
#include "common.h"

namespace sa {

constexpr int kShiftThreads = 256;

// Eight elements of a row as floats (VEC: one 16-byte load of bfloat16, two of float), and back.
template <typename T>
__device__ __forceinline__ void load8f(const T* p, float (&v)[8]) {
  if constexpr (sizeof(T) == 2) {
    const uint4 q = *reinterpret_cast<const uint4*>(p);
    const uint32_t w[4] = {q.x, q.y, q.z, q.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      v[2 * i] = __uint_as_float(w[i] << 16);
      v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
  } else {
    const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
    v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
    v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
  }
}
template <typename T>
__device__ __forceinline__ void store8f(T* p, const float (&v)[8]) {
  if constexpr (sizeof(T) == 2) {
    uint32_t w[4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
      w[i] = static_cast<uint32_t>(float_to_bf16(v[2 * i]).bits) | (static_cast<uint32_t>(float_to_bf16(v[2 * i + 1]).bits) << 16);
    *reinterpret_cast<uint4*>(p) = uint4{w[0], w[1], w[2], w[3]};
  } else {
    *reinterpret_cast<float4*>(p) = float4{v[0], v[1], v[2], v[3]};
    *reinterpret_cast<float4*>(p + 4) = float4{v[4], v[5], v[6], v[7]};
  }
}

// Grid (most tokens of a request, requests, pieces of the row).  The thread of a request's first token of the step
// that reads a channel's tail also moves it on to the request's last row: it alone touches it.
// VEC: channels per thread (8: rows, tails and weights are 16-byte aligned and D is a multiple of 8).
template <typename T, typename WT, int VEC>
__global__ __launch_bounds__(kShiftThreads) void token_shift_kernel(const T* __restrict__ h, int64_t h_stride,
                                                                    const WT* __restrict__ mu, int streams,
                                                                    float* __restrict__ tails, int64_t tail_stride,
                                                                    const int* __restrict__ seq_meta, T* __restrict__ out,
                                                                    int D) {
  const int* meta = seq_meta + 4 * blockIdx.y;
  const int slot = meta[0], first = meta[1], count = meta[2];
  const int j = blockIdx.x;
  const int d = (blockIdx.z * kShiftThreads + threadIdx.x) * VEC;
  if (j >= count || d >= D) return;
  const size_t t = static_cast<size_t>(first + j);
  float now[VEC], before[VEC];
  if constexpr (VEC == 8) load8f(h + t * h_stride + d, now);
  else now[0] = to_float(h[t * h_stride + d]);
  if (j > 0) {
    if constexpr (VEC == 8) load8f(h + (t - 1) * h_stride + d, before);
    else before[0] = to_float(h[(t - 1) * h_stride + d]);
  } else {
    float* tail = tails + static_cast<size_t>(slot) * tail_stride + d;
    const size_t last = static_cast<size_t>(first + count - 1);
    float next[VEC];
    if constexpr (VEC == 8) {
      load8f(tail, before);
      load8f(h + last * h_stride + d, next);
      store8f(tail, next);
    } else {
      before[0] = tail[0];
      next[0] = to_float(h[last * h_stride + d]);
      tail[0] = next[0];
    }
  }
  T* row = out + t * streams * D + d;
  for (int s = 0; s < streams; ++s) {
    float m[VEC], v[VEC];
    if constexpr (VEC == 8) load8f(mu + static_cast<size_t>(s) * D + d, m);
    else m[0] = to_float(mu[static_cast<size_t>(s) * D + d]);
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = fmaf(before[i] - now[i], m[i], now[i]);
    if constexpr (VEC == 8) store8f(row + static_cast<size_t>(s) * D, v);
    else row[static_cast<size_t>(s) * D] = from_float<T>(v[0]);
  }
}

// A wave takes 64 channels of kDecayTokens tokens: tanh(p) of the tokens goes through LDS, kDecayRank factors at a
// time, a lane sums its channel for all the tokens in the factors' order.  w is [rank, C]: a wave's loads of a factor
// are contiguous.
constexpr int kDecayTokens = 16;
constexpr int kDecayRank = 64;
template <typename WT>
__global__ __launch_bounds__(kWave) void low_rank_decay_kernel(const void* __restrict__ p, int p_dtype, int64_t p_stride,
                                                               const WT* __restrict__ w, const void* __restrict__ w0,
                                                               int w0_dtype, float* __restrict__ out, int T, int C,
                                                               int rank) {
  __shared__ __align__(16) float ts[kDecayTokens][kDecayRank];
  const int lane = threadIdx.x, c = blockIdx.x * kWave + lane, t0 = blockIdx.y * kDecayTokens;
  const int cc = c < C ? c : C - 1;
  float acc[kDecayTokens];
#pragma unroll
  for (int k = 0; k < kDecayTokens; ++k) acc[k] = 0.f;
  for (int r0 = 0; r0 < rank; r0 += kDecayRank) {
    __syncthreads();
    for (int e = lane; e < kDecayTokens * kDecayRank; e += kWave) {
      const int k = e / kDecayRank, r = e % kDecayRank;
      ts[k][r] = (t0 + k < T && r0 + r < rank) ? tanhf(load_f(p, p_dtype, static_cast<size_t>(t0 + k) * p_stride + r0 + r)) : 0.f;
    }
    __syncthreads();
    const int rn = rank - r0 < kDecayRank ? rank - r0 : kDecayRank;
    for (int r = 0; r < rn; r += 4) {
      float wv[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) wv[i] = r + i < rn ? to_float(w[static_cast<size_t>(r0 + r + i) * C + cc]) : 0.f;
#pragma unroll
      for (int k = 0; k < kDecayTokens; ++k) {
        const float4 x = *reinterpret_cast<const float4*>(&ts[k][r]);
        acc[k] = fmaf(x.x, wv[0], acc[k]);
        acc[k] = fmaf(x.y, wv[1], acc[k]);
        acc[k] = fmaf(x.z, wv[2], acc[k]);
        acc[k] = fmaf(x.w, wv[3], acc[k]);
      }
    }
  }
  if (c >= C) return;
  const float base = load_f(w0, w0_dtype, c);
#pragma unroll
  for (int k = 0; k < kDecayTokens; ++k)
    if (t0 + k < T) out[static_cast<size_t>(t0 + k) * C + c] = expf(-expf(acc[k] + base));
}

__global__ __launch_bounds__(256) void concat_rows_kernel(const float* __restrict__ x, const float* __restrict__ y,
                                                          void* __restrict__ out, int out_dtype, int D, int E) {
  const size_t t = blockIdx.x;
  const int d = blockIdx.y * 256 + threadIdx.x;
  if (d < D + E) store_f(out, out_dtype, t * (D + E) + d, d < D ? x[t * D + d] : y[t * E + d - D]);
}

}  // namespace sa

using namespace sa;

extern "C" int sa_token_shift(const void* h, int dtype, int64_t h_stride, const void* mu, int mu_dtype, int streams,
                              float* tails, int64_t tail_stride, const int* seq_meta, int num_seqs, int max_q_len,
                              void* out, int D, hipStream_t stream) {
  if (num_seqs == 0 || max_q_len == 0) return 0;
  SA_REQUIRE(num_seqs > 0 && num_seqs <= 65535 && max_q_len > 0 && D > 0 && streams > 0,
             "token_shift: bad sizes S=%d q=%d D=%d streams=%d", num_seqs, max_q_len, D, streams);
  SA_REQUIRE(h != nullptr && mu != nullptr && tails != nullptr && seq_meta != nullptr && out != nullptr,
             "token_shift: a null pointer");
  SA_REQUIRE(h_stride >= D && tail_stride >= D, "token_shift: rows or tails are shorter than the width %d", D);
  SA_REQUIRE((dtype == kF32 || dtype == kBF16) && (mu_dtype == kF32 || mu_dtype == kBF16), "token_shift: unknown dtype");
  auto aligned = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15u) == 0; };
  const bool vec = D % 8 == 0 && h_stride % 8 == 0 && tail_stride % 4 == 0 && aligned(h) && aligned(mu) && aligned(tails) &&
                   aligned(out);
#define SA_SHIFT(T, WT, V)                                                                                              \
  token_shift_kernel<T, WT, V><<<dim3(max_q_len, num_seqs, (D + kShiftThreads * V - 1) / (kShiftThreads * V)),          \
                                 kShiftThreads, 0, stream>>>(static_cast<const T*>(h), h_stride,                        \
                                                             static_cast<const WT*>(mu), streams, tails, tail_stride,   \
                                                             seq_meta, static_cast<T*>(out), D)
#define SA_SHIFT_W(T, V)                     \
  do {                                       \
    if (mu_dtype == kBF16) SA_SHIFT(T, bf16, V); \
    else SA_SHIFT(T, float, V);              \
  } while (0)
  if (dtype == kBF16) {
    if (vec) SA_SHIFT_W(bf16, 8);
    else SA_SHIFT_W(bf16, 1);
  } else {
    if (vec) SA_SHIFT_W(float, 8);
    else SA_SHIFT_W(float, 1);
  }
#undef SA_SHIFT_W
#undef SA_SHIFT
  return check_launch("token_shift");
}

extern "C" int sa_low_rank_decay(const void* p, int p_dtype, int64_t p_stride, const void* w, int w_dtype, const void* w0,
                                 int w0_dtype, float* out, int T, int C, int rank, hipStream_t stream) {
  if (T == 0) return 0;
  SA_REQUIRE(T > 0 && C > 0 && rank > 0 && p_stride >= rank, "low_rank_decay: bad sizes T=%d C=%d rank=%d", T, C, rank);
  SA_REQUIRE(p != nullptr && w != nullptr && w0 != nullptr && out != nullptr, "low_rank_decay: a null pointer");
  SA_REQUIRE((w_dtype == kF32 || w_dtype == kBF16) && (p_dtype == kF32 || p_dtype == kBF16) &&
                 (w0_dtype == kF32 || w0_dtype == kBF16),
             "low_rank_decay: unknown dtype");
  const dim3 grid((C + kWave - 1) / kWave, (T + kDecayTokens - 1) / kDecayTokens);
  SA_REQUIRE(grid.y <= 65535, "low_rank_decay: too many tokens");
  if (w_dtype == kBF16)
    low_rank_decay_kernel<bf16><<<grid, kWave, 0, stream>>>(p, p_dtype, p_stride, static_cast<const bf16*>(w), w0, w0_dtype,
                                                            out, T, C, rank);
  else
    low_rank_decay_kernel<float><<<grid, kWave, 0, stream>>>(p, p_dtype, p_stride, static_cast<const float*>(w), w0,
                                                             w0_dtype, out, T, C, rank);
  return check_launch("low_rank_decay");
}

extern "C" int sa_concat_rows(const float* x, const float* y, void* out, int out_dtype, int T, int D, int E,
                              hipStream_t stream) {
  if (T == 0) return 0;
  SA_REQUIRE(T > 0 && D > 0 && E > 0 && D + E <= 65535 * 256 && x != nullptr && y != nullptr && out != nullptr,
             "concat_rows: bad sizes T=%d D=%d E=%d", T, D, E);
  SA_REQUIRE(out_dtype == kF32 || out_dtype == kBF16, "concat_rows: unknown dtype %d", out_dtype);
  concat_rows_kernel<<<dim3(T, (D + E + 255) / 256), 256, 0, stream>>>(x, y, out, out_dtype, D, E);
  return check_launch("concat_rows");
}
