// What stands around the recurrence of a state-space mixer (one decay per head, queries and keys shared by groups of
// heads; the recurrence itself is linear_state.hip's):
//
//   ssm_inputs          a causal convolution per channel with a bias and silu, and per head the step size
//                       dt = softplus(p + dt_bias), the decay's logarithm l = -exp(A_log) dt and the decay exp(l)
//   gated_group_norm    (y * silu(z)) normed in equal groups of channels, times a weight per channel: the gate first
//
// A request's tokens of this step are rows first .. first + count - 1 (seq_meta [S, 4]: state slot, first row, count,
// position of the first); the convolution's last taps - 1 inputs of earlier steps are the slot's tail.  Convolution sums,
// step sizes, decays and the norm are 32-bit.
#include "api.h"
#include "common.h"

namespace sa {

constexpr int kSsmMaxTaps = 8;   // (at most kSsmTokens + 1: only a request's first tokens read its tail)
constexpr int kSsmTokens = 8;   // tokens that one thread of the convolution walks through

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 ssm_bf16x8;

__device__ inline void load8(const bf16* p, float (&v)[8]) {
  const ssm_bf16x8 x = *reinterpret_cast<const ssm_bf16x8*>(p);
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = static_cast<float>(x[e]);
}
__device__ inline void load8(const float* p, float (&v)[8]) {
  const float4 a = reinterpret_cast<const float4*>(p)[0], b = reinterpret_cast<const float4*>(p)[1];
  v[0] = a.x, v[1] = a.y, v[2] = a.z, v[3] = a.w, v[4] = b.x, v[5] = b.y, v[6] = b.z, v[7] = b.w;
}
__device__ inline void store8(bf16* p, const float (&v)[8]) {
  ssm_bf16x8 x;
#pragma unroll
  for (int e = 0; e < 8; ++e) x[e] = static_cast<__bf16>(v[e]);
  *reinterpret_cast<ssm_bf16x8*>(p) = x;
}
__device__ inline void store8(float* p, const float (&v)[8]) {
  reinterpret_cast<float4*>(p)[0] = float4{v[0], v[1], v[2], v[3]};
  reinterpret_cast<float4*>(p)[1] = float4{v[4], v[5], v[6], v[7]};
}

// z sigmoid(z): a result that is rounded to bfloat16 takes the hardware's exponential and reciprocal, a 32-bit one the
// library's.
template <typename T>
__device__ __forceinline__ float silu_for(float z) {
  if constexpr (sizeof(T) == 2) return z * __builtin_amdgcn_rcpf(1.f + __expf(-z));
  else return z / (1.f + expf(-z));
}

struct SsmInputs {
  int64_t row_stride, tail_stride;
  int x_at, dt_at, C, H, taps;
};

// gates [T, 3 H]: decays, step sizes, the decays' logarithms
template <typename T>
__device__ inline void ssm_gates(const T* proj, const SsmInputs& p, const void* dt_bias, const void* a_log, int vec_dtype,
                                 int row0, int rows, float* gates) {
  for (int i = threadIdx.x; i < rows * p.H; i += blockDim.x) {
    const int h = i % p.H;
    const size_t t = row0 + i / p.H;
    const float z = to_float(proj[t * p.row_stride + p.dt_at + h]) + load_f(dt_bias, vec_dtype, h);
    const float dt = z > 30.f ? z : log1pf(expf(z));
    const float l = -expf(load_f(a_log, vec_dtype, h)) * dt;
    float* g = gates + t * 3 * p.H;
    g[h] = expf(l);
    g[p.H + h] = dt;
    g[2 * p.H + h] = l;
  }
}

// A thread takes eight neighbouring channels of kSsmTokens consecutive tokens of a request, the last inputs in registers.
// The thread of a request's first tokens reads the channels' tails and afterwards moves them on to the step's last inputs:
// it alone touches them.  taps_by_tap [N][C].  The last blockIdx.z computes the gates.
template <typename T, typename WT, int N>
__global__ __launch_bounds__(kWave) void ssm_inputs_kernel(const T* __restrict__ proj, SsmInputs p,
                                                           const WT* __restrict__ taps_by_tap, const WT* __restrict__ bias,
                                                           const void* __restrict__ dt_bias, const void* __restrict__ a_log,
                                                           int vec_dtype, float* __restrict__ tails,
                                                           const int* __restrict__ seq_meta, T* __restrict__ y,
                                                           float* __restrict__ gates) {
  const int* meta = seq_meta + 4 * blockIdx.y;
  const int slot = meta[0], first = meta[1], count = meta[2];
  const int j0 = blockIdx.x * kSsmTokens;
  if (j0 >= count) return;
  const int jn = count - j0 < kSsmTokens ? count - j0 : kSsmTokens;
  if (blockIdx.z == gridDim.z - 1) {
    ssm_gates(proj, p, dt_bias, a_log, vec_dtype, first + j0, jn, gates);
    return;
  }
  const int c = (blockIdx.z * kWave + threadIdx.x) * 8;
  if (c >= p.C) return;
  float w[N][8], b[8], win[N][8];   // win[i]: the input under tap i
  float* tail = tails + static_cast<size_t>(slot) * p.tail_stride;
#pragma unroll
  for (int i = 0; i < N; ++i) load8(taps_by_tap + static_cast<size_t>(i) * p.C + c, w[i]);
  load8(bias + c, b);
  const T* col = proj + static_cast<size_t>(first) * p.row_stride + p.x_at + c;
#pragma unroll
  for (int i = 1; i < N; ++i) {   // the N - 1 inputs before j0, one place further on
    const int j = j0 - N + i;
    if (j >= 0) load8(col + static_cast<size_t>(j) * p.row_stride, win[i]);
    else load8(tail + static_cast<size_t>(N - 1 + j) * p.C + c, win[i]);
  }
  if (j0 == 0) {
    // the new tail: the step's last N - 1 inputs, the older of them from the tail as it was (its entries are in win)
#pragma unroll
    for (int i = 0; i + 1 < N; ++i) {
      const int j = count - (N - 1) + i;
      float v[8];
      if (j >= 0) {
        load8(col + static_cast<size_t>(j) * p.row_stride, v);
      } else {
#pragma unroll
        for (int k = 1; k < N; ++k)
          if (k == N + j)
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] = win[k][e];
      }
      store8(tail + static_cast<size_t>(i) * p.C + c, v);
    }
  }
  float in[kSsmTokens][8];
#pragma unroll
  for (int j = 0; j < kSsmTokens; ++j) load8(col + static_cast<size_t>(j0 + (j < jn ? j : jn - 1)) * p.row_stride, in[j]);
#pragma unroll
  for (int j = 0; j < kSsmTokens; ++j) {
    if (j >= jn) break;   // (uniform)
    float acc[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      acc[e] = 0.f;
#pragma unroll
      for (int i = 0; i < N; ++i) {
        const int at = j - (N - 1) + i;   // before j0: win[N + at]
        acc[e] = fmaf(w[i][e], at >= 0 ? in[at >= 0 ? at : 0][e] : win[at < 0 ? N + at : 0][e], acc[e]);
      }
      acc[e] = silu_for<T>(acc[e] + b[e]);
    }
    store8(y + static_cast<size_t>(first + j0 + j) * p.C + c, acc);
  }
}

// Any number of taps and channels: a thread takes one channel of kSsmTokens tokens; the tails as above.
template <typename T>
__global__ __launch_bounds__(kWave) void ssm_inputs_any_kernel(const T* __restrict__ proj, SsmInputs p,
                                                               const void* __restrict__ taps_by_tap,
                                                               const void* __restrict__ bias, int taps_dtype,
                                                               const void* __restrict__ dt_bias,
                                                               const void* __restrict__ a_log, int vec_dtype,
                                                               float* __restrict__ tails, const int* __restrict__ seq_meta,
                                                               T* __restrict__ y, float* __restrict__ gates) {
  const int* meta = seq_meta + 4 * blockIdx.y;
  const int slot = meta[0], first = meta[1], count = meta[2];
  const int j0 = blockIdx.x * kSsmTokens, n = p.taps;
  if (j0 >= count) return;
  const int jn = count - j0 < kSsmTokens ? count - j0 : kSsmTokens;
  if (blockIdx.z == gridDim.z - 1) {
    ssm_gates(proj, p, dt_bias, a_log, vec_dtype, first + j0, jn, gates);
    return;
  }
  const int c = blockIdx.z * kWave + threadIdx.x;
  if (c >= p.C) return;
  float* tail = tails + static_cast<size_t>(slot) * p.tail_stride;
  const T* col = proj + static_cast<size_t>(first) * p.row_stride + p.x_at + c;
  for (int j = j0; j < j0 + jn; ++j) {
    float acc = 0.f;
    for (int i = 0; i < n; ++i) {
      const int jj = j - (n - 1) + i;
      const float u = jj >= 0 ? to_float(col[static_cast<size_t>(jj) * p.row_stride])
                              : tail[static_cast<size_t>(n - 1 + jj) * p.C + c];
      acc = fmaf(load_f(taps_by_tap, taps_dtype, static_cast<size_t>(i) * p.C + c), u, acc);
    }
    acc += load_f(bias, taps_dtype, c);
    y[static_cast<size_t>(first + j) * p.C + c] = from_float<T>(silu_for<T>(acc));
  }
  if (j0 > 0) return;
  for (int i = 0; i < n - 1; ++i) {   // (old entries are read at places that have not been written yet)
    const int j = count - (n - 1) + i;
    tail[static_cast<size_t>(i) * p.C + c] =
        j >= 0 ? to_float(col[static_cast<size_t>(j) * p.row_stride]) : tail[static_cast<size_t>(n - 1 + j) * p.C + c];
  }
}

// A workgroup of NT threads per (token, group).  NP > 0: the group's entries are held in registers, NP pieces of VEC a thread; 0: they
// are read twice.
template <typename T, int VEC, int NP, int NT>
__global__ __launch_bounds__(NT) void gated_group_norm_kernel(const float* __restrict__ y, int64_t y_stride,
                                                               const T* __restrict__ z, int64_t z_stride,
                                                               const void* __restrict__ w, int w_dtype, float eps,
                                                               T* __restrict__ out, int64_t out_stride, int size) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, c0 = blockIdx.y * size;
  const float* yr = y + static_cast<size_t>(t) * y_stride + c0;
  const T* zr = z + static_cast<size_t>(t) * z_stride + c0;
  T* orow = out + static_cast<size_t>(t) * out_stride + c0;
  auto gated = [&](float yv, T zv) { return yv * silu_for<T>(to_float(zv)); };
  float ss = 0.f;
  if constexpr (NP == 0) {
    for (int d = threadIdx.x; d < size; d += NT) {
      const float v = gated(yr[d], zr[d]);
      ss = fmaf(v, v, ss);
    }
    const float r = 1.f / sqrtf((NT == kWave ? wave_sum(ss) : block_sum(ss, scratch)) / static_cast<float>(size) + eps);
    for (int d = threadIdx.x; d < size; d += NT)
      orow[d] = from_float<T>(gated(yr[d], zr[d]) * r * load_f(w, w_dtype, c0 + d));
  } else {
    float v[NP][VEC];
    float yv[NP][VEC];
    T zv[NP][VEC];
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const int d = (threadIdx.x + i * NT) * VEC;
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        yv[i][e] = 0.f;
        zv[i][e] = from_float<T>(0.f);
      }
      if (d < size) {
        if constexpr (VEC == 4) {
          *reinterpret_cast<float4*>(yv[i]) = *reinterpret_cast<const float4*>(yr + d);
          if constexpr (sizeof(T) == 2) *reinterpret_cast<uint2*>(zv[i]) = *reinterpret_cast<const uint2*>(zr + d);
          else *reinterpret_cast<uint4*>(zv[i]) = *reinterpret_cast<const uint4*>(zr + d);
        } else {
          yv[i][0] = yr[d];
          zv[i][0] = zr[d];
        }
      }
    }
#pragma unroll
    for (int i = 0; i < NP; ++i)
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        v[i][e] = gated(yv[i][e], zv[i][e]);
        ss = fmaf(v[i][e], v[i][e], ss);
      }
    const float r = 1.f / sqrtf((NT == kWave ? wave_sum(ss) : block_sum(ss, scratch)) / static_cast<float>(size) + eps);
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const int d = (threadIdx.x + i * NT) * VEC;
      if (d >= size) continue;
      T o[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) o[e] = from_float<T>(v[i][e] * r * load_f(w, w_dtype, c0 + d + e));
      if constexpr (VEC == 4 && sizeof(T) == 2) *reinterpret_cast<uint2*>(orow + d) = *reinterpret_cast<const uint2*>(o);
      else if constexpr (VEC == 4) *reinterpret_cast<uint4*>(orow + d) = *reinterpret_cast<const uint4*>(o);
      else orow[d] = o[0];
    }
  }
}

template <typename T>
static void launch_gated_group_norm(const float* y, int64_t y_stride, const void* z_, int64_t z_stride, const void* w,
                                    int w_dtype, float eps, void* out_, int64_t out_stride, int T_, int groups, int size,
                                    hipStream_t stream) {
  const T* z = static_cast<const T*>(z_);
  T* out = static_cast<T*>(out_);
  const dim3 grid(T_, groups);
#define SA_GROUP_NORM(VEC, NP, NT) \
  gated_group_norm_kernel<T, VEC, NP, NT><<<grid, NT, 0, stream>>>(y, y_stride, z, z_stride, w, w_dtype, eps, out, out_stride, size)
  auto aligned = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool vec = size % 4 == 0 && y_stride % 4 == 0 && z_stride % 4 == 0 && out_stride % 4 == 0 && aligned(y) && aligned(z) &&
                   aligned(out);
  if (vec && size <= 256) SA_GROUP_NORM(4, 1, 64);
  else if (vec && size <= 512) SA_GROUP_NORM(4, 2, 64);
  else if (vec && size <= 1024) SA_GROUP_NORM(4, 1, 256);
  else if (vec && size <= 2048) SA_GROUP_NORM(4, 2, 256);
  else if (vec && size <= 4096) SA_GROUP_NORM(4, 4, 256);
  else if (vec && size <= 8192) SA_GROUP_NORM(4, 8, 256);
  else if (!vec && size <= 512) SA_GROUP_NORM(1, 2, 256);
  else SA_GROUP_NORM(1, 0, 256);
#undef SA_GROUP_NORM
}

template <typename T, typename WT, int N>
static void launch_ssm_inputs(const void* proj, const SsmInputs& p, const void* taps, const void* bias, const void* dt_bias,
                              const void* a_log, int vec_dtype, float* tails, const int* seq_meta, int num_seqs,
                              int max_q_len, void* y, float* gates, hipStream_t stream) {
  const int cz = (p.C / 8 + kWave - 1) / kWave + 1;
  const dim3 grid((max_q_len + kSsmTokens - 1) / kSsmTokens, num_seqs, cz);
  ssm_inputs_kernel<T, WT, N><<<grid, kWave, 0, stream>>>(static_cast<const T*>(proj), p, static_cast<const WT*>(taps),
                                                          static_cast<const WT*>(bias), dt_bias, a_log, vec_dtype, tails,
                                                          seq_meta, static_cast<T*>(y), gates);
}

}  // namespace sa

using namespace sa;

extern "C" int sa_ssm_inputs(const void* proj, int dtype, int64_t row_stride, int x_at, int dt_at, int C, const void* taps,
                             const void* bias, int taps_dtype, int num_taps, const void* dt_bias, const void* a_log,
                             int vec_dtype, float* tails, int64_t tail_stride, const int* seq_meta,
                             int num_seqs, int max_q_len, void* y, float* gates, int H, hipStream_t stream) {
  if (num_seqs == 0 || max_q_len == 0) return 0;
  SA_REQUIRE(num_seqs > 0 && num_seqs <= 65535 && max_q_len > 0 && C > 0 && H > 0 && x_at >= 0 && dt_at >= 0 &&
                 row_stride >= x_at + static_cast<int64_t>(C) && row_stride >= dt_at + static_cast<int64_t>(H),
             "ssm_inputs: bad sizes S=%d q=%d C=%d H=%d", num_seqs, max_q_len, C, H);
  SA_REQUIRE(num_taps >= 1 && num_taps <= kSsmMaxTaps, "ssm_inputs: %d taps (1 to %d)", num_taps, kSsmMaxTaps);
  SA_REQUIRE(proj != nullptr && taps != nullptr && bias != nullptr && dt_bias != nullptr && a_log != nullptr &&
                 seq_meta != nullptr && y != nullptr && gates != nullptr && (num_taps == 1 || tails != nullptr) &&
                 tail_stride >= static_cast<int64_t>(num_taps - 1) * C,
             "ssm_inputs: a null pointer or tails that are too short");
  SA_REQUIRE((dtype == kF32 || dtype == kBF16) && (taps_dtype == kF32 || taps_dtype == kBF16) &&
                 (vec_dtype == kF32 || vec_dtype == kBF16),
             "ssm_inputs: unknown dtype");
  SA_REQUIRE((C + kWave - 1) / kWave < 65535, "ssm_inputs: too many channels");
  SsmInputs p;
  p.row_stride = row_stride, p.tail_stride = tail_stride, p.x_at = x_at, p.dt_at = dt_at, p.C = C, p.H = H, p.taps = num_taps;
  auto aligned = [](const void* q) { return reinterpret_cast<uintptr_t>(q) % 16 == 0; };
  const bool pieces = num_taps >= 2 && num_taps <= 4 && C % 8 == 0 && x_at % 8 == 0 && row_stride % 8 == 0 && tail_stride % 4 == 0 &&
                      aligned(proj) && aligned(taps) && aligned(bias) && aligned(tails) && aligned(y);
  if (!pieces) {
    const dim3 grid((max_q_len + kSsmTokens - 1) / kSsmTokens, num_seqs, (C + kWave - 1) / kWave + 1);
    if (dtype == kBF16)
      ssm_inputs_any_kernel<bf16><<<grid, kWave, 0, stream>>>(static_cast<const bf16*>(proj), p, taps, bias, taps_dtype, dt_bias,
                                                              a_log, vec_dtype, tails, seq_meta, static_cast<bf16*>(y), gates);
    else
      ssm_inputs_any_kernel<float><<<grid, kWave, 0, stream>>>(static_cast<const float*>(proj), p, taps, bias, taps_dtype, dt_bias,
                                                               a_log, vec_dtype, tails, seq_meta, static_cast<float*>(y), gates);
    return check_launch("ssm_inputs");
  }
#define SA_SSM_TAPS(T_, W_)                                                                                            \
  do {                                                                                                                 \
    if (num_taps == 2) launch_ssm_inputs<T_, W_, 2>(proj, p, taps, bias, dt_bias, a_log, vec_dtype, tails, seq_meta, num_seqs, \
                                                    max_q_len, y, gates, stream);                                      \
    else if (num_taps == 3) launch_ssm_inputs<T_, W_, 3>(proj, p, taps, bias, dt_bias, a_log, vec_dtype, tails, seq_meta,   \
                                                         num_seqs, max_q_len, y, gates, stream);                       \
    else launch_ssm_inputs<T_, W_, 4>(proj, p, taps, bias, dt_bias, a_log, vec_dtype, tails, seq_meta, num_seqs, max_q_len, \
                                      y, gates, stream);                                                               \
  } while (0)
  if (dtype == kBF16) {
    if (taps_dtype == kBF16) SA_SSM_TAPS(bf16, bf16);
    else SA_SSM_TAPS(bf16, float);
  } else {
    if (taps_dtype == kBF16) SA_SSM_TAPS(float, bf16);
    else SA_SSM_TAPS(float, float);
  }
#undef SA_SSM_TAPS
  return check_launch("ssm_inputs");
}

extern "C" int sa_gated_group_norm(const float* y, int64_t y_stride, const void* z, int dtype, int64_t z_stride, const void* w,
                                   int w_dtype, float eps, void* out, int groups, int64_t out_stride, int T, int width,
                                   hipStream_t stream) {
  if (T == 0) return 0;
  SA_REQUIRE(T > 0 && groups > 0 && groups <= 65535 && width > 0 && width % groups == 0,
             "gated_group_norm: bad sizes T=%d, %d channels in %d groups", T, width, groups);
  SA_REQUIRE(y != nullptr && z != nullptr && w != nullptr && out != nullptr && y_stride >= width && z_stride >= width &&
                 out_stride >= width,
             "gated_group_norm: a null pointer or rows that are too short");
  SA_REQUIRE((dtype == kF32 || dtype == kBF16) && (w_dtype == kF32 || w_dtype == kBF16), "gated_group_norm: unknown dtype");
  if (dtype == kBF16)
    launch_gated_group_norm<bf16>(y, y_stride, z, z_stride, w, w_dtype, eps, out, out_stride, T, groups, width / groups, stream);
  else
    launch_gated_group_norm<float>(y, y_stride, z, z_stride, w, w_dtype, eps, out, out_stride, T, groups, width / groups, stream);
  return check_launch("gated_group_norm");
}
