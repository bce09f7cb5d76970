// What a mixer with a token shift and data-dependent decays reads, and the rows of a looped pass:
//
//   token_shift_kernel     out[t, s, :] = h[t] + (h[t - 1] - h[t]) * mu[s, :]   for every stream s of a mixer's input
//   low_rank_decay_kernel  a[t, c] = exp(-exp(sum_r w[c, r] tanh(p[t, r]) + w0[c]))
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

// 32-bit weights [C, rank], or bfloat16 ones as rows: a wave takes 64 channels of kDecayTokens tokens; tanh(p) of the
// tokens goes through LDS, kDecayRank factors at a time, a lane sums its channel for all the tokens in the factors' order.
constexpr int kDecayTokens = 16;
constexpr int kDecayRank = 64;
template <typename WT>
__global__ __launch_bounds__(kWave) void low_rank_decay_kernel(const void* __restrict__ p, int p_dtype, int64_t p_stride,
                                                               const WT* __restrict__ w, const void* __restrict__ w0,
                                                               int w0_dtype, float* __restrict__ out, int T, int C,
                                                               int rank) {
  __shared__ __align__(16) float ts[kDecayTokens][kDecayRank];
  const int lane = threadIdx.x, c = blockIdx.x * kWave + lane, t0 = blockIdx.y * kDecayTokens;
  const WT* row = w + static_cast<size_t>(c < C ? c : C - 1) * rank;
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
    for (int r = 0; r < rn; ++r) {
      const float wv = to_float(row[r0 + r]);
#pragma unroll
      for (int k = 0; k < kDecayTokens; ++k) acc[k] = fmaf(ts[k][r], wv, acc[k]);
    }
  }
  if (c >= C) return;
  const float base = load_f(w0, w0_dtype, c);
#pragma unroll
  for (int k = 0; k < kDecayTokens; ++k)
    if (t0 + k < T) out[static_cast<size_t>(t0 + k) * C + c] = expf(-expf(acc[k] + base));
}

// bfloat16 weights in MFMA operand tiles ([C / 16][rank / 32][64][8], zeros beyond C and rank): a wave takes 16 tokens and
// `tiles` tiles of 16 channels.  tanh(p) goes in as three bfloat16 numbers (its rounding, the rounding of what that leaves,
// and the rest: all 24 bits), so that the sum is that of 32-bit factors; a lane computes the eight entries of every 32
// that its operand holds.
typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;
constexpr int kDecayChunks = 2;   // chunks of 32 factors whose tanh a wave holds at a time
template <typename PT, typename BT, bool VEC>
__global__ __launch_bounds__(256) void low_rank_decay_tiled_kernel(const PT* __restrict__ p, int64_t p_stride,
                                                                   const bf16* __restrict__ w, const BT* __restrict__ w0,
                                                                   float* __restrict__ out, int T, int C, int rank,
                                                                   int tiles) {
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
  const int r = lane % 16, kq = lane / 16;
  const int t = blockIdx.y * 16 + r, tc = t < T ? t : T - 1;
  const int chunks = (rank + 31) / 32, all = (C + 15) / 16;
  const int n0 = (blockIdx.x * 4 + wave) * tiles, n1 = n0 + tiles < all ? n0 + tiles : all;
  if (n0 >= all) return;   // (a whole wave; there are no barriers)
  bf16x8 hi[kDecayChunks], mid[kDecayChunks], lo[kDecayChunks];
  auto factors = [&](int c0) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < kDecayChunks; ++u) {
      const int k0 = (c0 + u) * 32 + kq * 8;
      const PT* src = p + static_cast<size_t>(tc) * p_stride + k0;
      float xs[8];
      if (VEC && k0 + 8 <= rank) {
        load8f(src, xs);
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) xs[j] = k0 + j < rank ? to_float(src[j]) : 0.f;
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float x = xs[j];
        // tanh by the hardware's exponential: 1 - 2 / (e^(2x) + 1), and x (1 - x^2 / 3) where that cancels
        const float y = 1.f - 2.f * __builtin_amdgcn_rcpf(__expf(2.f * x) + 1.f);
        const float th = fabsf(x) < 0.02f ? x * fmaf(x * x, -1.f / 3.f, 1.f) : y;
        hi[u][j] = static_cast<__bf16>(th);
        const float rest = th - static_cast<float>(hi[u][j]);
        mid[u][j] = static_cast<__bf16>(rest);
        lo[u][j] = static_cast<__bf16>(rest - static_cast<float>(mid[u][j]));
      }
    }
  };
  if (chunks <= kDecayChunks) factors(0);   // (held for all of the wave's channels)
  // one pass holds the sums of up to 4 channel tiles
  for (int nb = n0; nb < n1; nb += 4) {
    floatx4 acc[4];   // (from the channels' constants)
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int v = 0; v < 4; ++v) {
        const int c = (nb + i < n1 ? nb + i : n1 - 1) * 16 + kq * 4 + v;
        acc[i][v] = to_float(w0[c < C ? c : C - 1]);
      }
    for (int c0 = 0; c0 < chunks; c0 += kDecayChunks) {
      bf16x8 wv[4][kDecayChunks];
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int u = 0; u < kDecayChunks; ++u) {
          const int tile = nb + i < n1 ? nb + i : n1 - 1, ch = c0 + u < chunks ? c0 + u : chunks - 1;
          wv[i][u] = *reinterpret_cast<const bf16x8*>(w + (static_cast<size_t>(tile) * chunks + ch) * 512 + lane * 8);
        }
      if (chunks > kDecayChunks) factors(c0);
#pragma unroll
      for (int u = 0; u < kDecayChunks; ++u) {
        if (c0 + u >= chunks) break;   // (uniform)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[i][u], hi[u], acc[i], 0, 0, 0);
          acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[i][u], mid[u], acc[i], 0, 0, 0);
          acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[i][u], lo[u], acc[i], 0, 0, 0);
        }
      }
    }
    // lane: token r, channels 4 kq .. of every tile
    if (t >= T) continue;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (nb + i >= n1) break;
      const int c = (nb + i) * 16 + kq * 4;
      float* dst = out + static_cast<size_t>(t) * C + c;
      float a[4];
#pragma unroll
      for (int v = 0; v < 4; ++v) a[v] = c + v < C ? __expf(-__expf(acc[i][v])) : 0.f;
      if (c + 4 <= C && C % 4 == 0) {
        *reinterpret_cast<float4*>(dst) = float4{a[0], a[1], a[2], a[3]};
      } else {
#pragma unroll
        for (int v = 0; v < 4; ++v)
          if (c + v < C) dst[v] = a[v];
      }
    }
  }
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

extern "C" int sa_low_rank_decay(const void* p, int p_dtype, int64_t p_stride, const void* w, int w_dtype, int tiled,
                                 const void* w0, int w0_dtype, float* out, int T, int C, int rank, hipStream_t stream) {
  if (T == 0) return 0;
  SA_REQUIRE(T > 0 && C > 0 && rank > 0 && p_stride >= rank, "low_rank_decay: bad sizes T=%d C=%d rank=%d", T, C, rank);
  SA_REQUIRE(p != nullptr && w != nullptr && w0 != nullptr && out != nullptr, "low_rank_decay: a null pointer");
  SA_REQUIRE((w_dtype == kF32 || w_dtype == kBF16) && (p_dtype == kF32 || p_dtype == kBF16) &&
                 (w0_dtype == kF32 || w0_dtype == kBF16),
             "low_rank_decay: unknown dtype");
  if (tiled) {
    SA_REQUIRE(w_dtype == kBF16, "low_rank_decay: tiled weights are bfloat16");
    // a wave takes one tile of channels while there are few tokens, up to eight when there are many (their tanh is shared)
    const int tt = (T + 15) / 16, all = (C + 15) / 16;
    const int64_t units = static_cast<int64_t>(tt) * all;
    const int tiles = units >= 8192 ? 8 : units >= 4096 ? 4 : 1;
    const dim3 grid((all + 4 * tiles - 1) / (4 * tiles), tt);
    SA_REQUIRE(grid.y <= 65535, "low_rank_decay: too many tokens");
    const bool vec = (reinterpret_cast<uintptr_t>(p) & 15u) == 0 && p_stride % 8 == 0;
#define SA_DECAY(PT, BT, V)                                                                                               \
  low_rank_decay_tiled_kernel<PT, BT, V><<<grid, 256, 0, stream>>>(static_cast<const PT*>(p), p_stride,                    \
                                                                   static_cast<const bf16*>(w), static_cast<const BT*>(w0), \
                                                                   out, T, C, rank, tiles)
#define SA_DECAY_B(PT, V)                      \
  do {                                         \
    if (w0_dtype == kBF16) SA_DECAY(PT, bf16, V); \
    else SA_DECAY(PT, float, V);               \
  } while (0)
    if (p_dtype == kBF16 && vec) SA_DECAY_B(bf16, true);
    else if (p_dtype == kBF16) SA_DECAY_B(bf16, false);
    else SA_DECAY_B(float, false);
#undef SA_DECAY_B
#undef SA_DECAY
    return check_launch("low_rank_decay");
  }
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
