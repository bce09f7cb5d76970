// A residual of several parallel streams x_1 .. x_S (hyper-connections).  A part reads a weighted sum of the streams and
// its result goes back into all of them, which are mixed at the same time:
//
//   x_t <- sum_s mix[s, t] x_s + out[t] y          (all streams at once, from the old ones)
//   u = sum_s in[s] x_s,  z = u / sqrt(mean(u^2) + eps) * w      what the next part reads
//
// Both in one pass over a token's streams: the update of one part and the read and norm of the next.  Streams, sums and
// the norm are 32-bit; y and z have the activation type.  The streams may be read where they all are one row (a stream
// stride of 0: the embedding's output) and are then written to memory of their own.
#include "api.h"
#include "common.h"

namespace sa {

constexpr int kMaxStreams = 16;

struct Streams {
  int64_t x_row, x_stream, y_stride;
  int S, planes, T, D;
  float eps;
};

// y of a product whose cuts of K are not added up yet: their sum in order, rounded as the product's own sum would be.
__device__ inline float planes_sum(const float* planes, int count, size_t plane, size_t at) {
  float v = planes[at];
  for (int p = 1; p < count; ++p) v += planes[static_cast<size_t>(p) * plane + at];
  return to_float(float_to_bf16(v));
}

// A workgroup per token; a thread holds NP pieces of four neighbouring entries of every stream.  T: activation type, WT:
// the norm weight's type, S: number of streams.
template <typename T, typename WT, int S, int NT, int NP>
__global__ __launch_bounds__(NT) void streams_kernel(const float* x, Streams p, float* h, const void* __restrict__ y_,
                                                     const float* __restrict__ mix, const float* __restrict__ out_w,
                                                     const float* __restrict__ in_w, const WT* __restrict__ w,
                                                     const int* __restrict__ rows, T* __restrict__ z) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, tid = threadIdx.x, D = p.D;
  const size_t row = rows != nullptr ? rows[t] : t;
  const float* xr = x + row * p.x_row;
  float4 xv[NP][S], yv[NP];
#pragma unroll
  for (int i = 0; i < NP; ++i) {
    const int d = (tid + i * NT) * 4;
#pragma unroll
    for (int s = 0; s < S; ++s)
      xv[i][s] = d < D ? *reinterpret_cast<const float4*>(xr + s * p.x_stream + d) : float4{0.f, 0.f, 0.f, 0.f};
    yv[i] = float4{0.f, 0.f, 0.f, 0.f};
    if (y_ != nullptr && d < D) {
      if (p.planes > 0) {
        const float* yp = static_cast<const float*>(y_);
        const size_t plane = static_cast<size_t>(p.T) * D, at = static_cast<size_t>(t) * D + d;
        float4 v = *reinterpret_cast<const float4*>(yp + at);
        for (int k = 1; k < p.planes; ++k) {
          const float4 a = *reinterpret_cast<const float4*>(yp + k * plane + at);
          v.x += a.x, v.y += a.y, v.z += a.z, v.w += a.w;
        }
        yv[i] = float4{to_float(float_to_bf16(v.x)), to_float(float_to_bf16(v.y)), to_float(float_to_bf16(v.z)),
                       to_float(float_to_bf16(v.w))};
      } else {
        const T* yp = static_cast<const T*>(y_) + static_cast<size_t>(t) * p.y_stride + d;
        T e[4];
        if constexpr (sizeof(T) == 2) *reinterpret_cast<uint2*>(e) = *reinterpret_cast<const uint2*>(yp);
        else *reinterpret_cast<uint4*>(e) = *reinterpret_cast<const uint4*>(yp);
        yv[i] = float4{to_float(e[0]), to_float(e[1]), to_float(e[2]), to_float(e[3])};
      }
    }
  }
  if (y_ != nullptr) {
    float* hr = h + static_cast<size_t>(t) * S * D;
    float m[S][S], o[S];
#pragma unroll
    for (int s = 0; s < S; ++s) {
      o[s] = out_w[s];
#pragma unroll
      for (int q = 0; q < S; ++q) m[s][q] = mix[s * S + q];
    }
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const int d = (tid + i * NT) * 4;
      float4 nv[S];
#pragma unroll
      for (int q = 0; q < S; ++q) {
        float4 a{o[q] * yv[i].x, o[q] * yv[i].y, o[q] * yv[i].z, o[q] * yv[i].w};
#pragma unroll
        for (int s = 0; s < S; ++s) {
          a.x = fmaf(m[s][q], xv[i][s].x, a.x);
          a.y = fmaf(m[s][q], xv[i][s].y, a.y);
          a.z = fmaf(m[s][q], xv[i][s].z, a.z);
          a.w = fmaf(m[s][q], xv[i][s].w, a.w);
        }
        nv[q] = a;
      }
#pragma unroll
      for (int q = 0; q < S; ++q) {
        xv[i][q] = nv[q];
        if (d < D) *reinterpret_cast<float4*>(hr + static_cast<size_t>(q) * D + d) = nv[q];
      }
    }
  }
  if (in_w == nullptr) return;
  float4 u[NP], wv[NP];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NP; ++i) {
    const int d = (tid + i * NT) * 4;
    u[i] = float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < S; ++s) {
      const float c = in_w[s];
      u[i].x = fmaf(c, xv[i][s].x, u[i].x);
      u[i].y = fmaf(c, xv[i][s].y, u[i].y);
      u[i].z = fmaf(c, xv[i][s].z, u[i].z);
      u[i].w = fmaf(c, xv[i][s].w, u[i].w);
    }
    ss = fmaf(u[i].x, u[i].x, ss);
    ss = fmaf(u[i].y, u[i].y, ss);
    ss = fmaf(u[i].z, u[i].z, ss);
    ss = fmaf(u[i].w, u[i].w, ss);
    wv[i] = float4{1.f, 1.f, 1.f, 1.f};
    if (w != nullptr && d < D) wv[i] = float4{to_float(w[d]), to_float(w[d + 1]), to_float(w[d + 2]), to_float(w[d + 3])};
  }
  float r = 1.f;
  if (w != nullptr) r = 1.f / sqrtf(block_sum(ss, scratch) / static_cast<float>(D) + p.eps);
#pragma unroll
  for (int i = 0; i < NP; ++i) {
    const int d = (tid + i * NT) * 4;
    if (d >= D) continue;
    T e[4] = {from_float<T>(u[i].x * r * wv[i].x), from_float<T>(u[i].y * r * wv[i].y), from_float<T>(u[i].z * r * wv[i].z),
              from_float<T>(u[i].w * r * wv[i].w)};
    T* zp = z + static_cast<size_t>(t) * D + d;
    if constexpr (sizeof(T) == 2) *reinterpret_cast<uint2*>(zp) = *reinterpret_cast<const uint2*>(e);
    else *reinterpret_cast<uint4*>(zp) = *reinterpret_cast<const uint4*>(e);
  }
}

// Any number of streams up to kMaxStreams and any width: entry by entry, the sums read waiting in LDS for the norm.
__global__ __launch_bounds__(256) void streams_any_kernel(const float* x, Streams p, float* h, const void* __restrict__ y,
                                                          int y_dtype, const float* __restrict__ mix,
                                                          const float* __restrict__ out_w, const float* __restrict__ in_w,
                                                          const void* __restrict__ w, int w_dtype,
                                                          const int* __restrict__ rows, void* __restrict__ z, int z_dtype) {
  extern __shared__ float u_s[];
  __shared__ float scratch[16];
  const int t = blockIdx.x, D = p.D, S = p.S;
  const size_t row = rows != nullptr ? rows[t] : t;
  const float* xr = x + row * p.x_row;
  float ss = 0.f;
  for (int d = threadIdx.x; d < D; d += 256) {
    float xv[kMaxStreams];
#pragma unroll
    for (int s = 0; s < kMaxStreams; ++s) xv[s] = s < S ? xr[s * p.x_stream + d] : 0.f;
    float yv = 0.f;
    if (y != nullptr)
      yv = p.planes > 0 ? planes_sum(static_cast<const float*>(y), p.planes, static_cast<size_t>(p.T) * D,
                                     static_cast<size_t>(t) * D + d)
                        : load_f(y, y_dtype, static_cast<size_t>(t) * p.y_stride + d);
    float u = 0.f;
    for (int q = 0; q < S; ++q) {
      float v;
      if (y != nullptr) {
        v = out_w[q] * yv;
#pragma unroll
        for (int s = 0; s < kMaxStreams; ++s)
          if (s < S) v = fmaf(mix[s * S + q], xv[s], v);
        h[(static_cast<size_t>(t) * S + q) * D + d] = v;
      } else {
        v = xr[q * p.x_stream + d];
      }
      if (in_w != nullptr) u = fmaf(in_w[q], v, u);
    }
    if (in_w != nullptr) {
      u_s[d] = u;
      ss = fmaf(u, u, ss);
    }
  }
  if (in_w == nullptr) return;
  float r = 1.f;
  if (w != nullptr) r = 1.f / sqrtf(block_sum(ss, scratch) / static_cast<float>(D) + p.eps);
  for (int d = threadIdx.x; d < D; d += 256)   // (a thread reads what it wrote itself)
    store_f(z, z_dtype, static_cast<size_t>(t) * D + d, w != nullptr ? u_s[d] * r * load_f(w, w_dtype, d) : u_s[d]);
}

template <typename T, typename WT, int S>
static void launch_streams(const float* x, const Streams& p, float* h, const void* y, const float* mix, const float* out_w,
                           const float* in_w, const void* w, const int* rows, void* z, hipStream_t stream) {
#define SA_STREAMS(NT, NP)                                                                                          \
  streams_kernel<T, WT, S, NT, NP><<<p.T, NT, 0, stream>>>(x, p, h, y, mix, out_w, in_w, static_cast<const WT*>(w), rows, \
                                                           static_cast<T*>(z))
  const int pieces = p.D / 4;
  if (pieces <= 256) SA_STREAMS(256, 1);
  else if (pieces > 1024) SA_STREAMS(1024, 2);
  else if (p.T <= 256 && pieces > 512) SA_STREAMS(1024, 1);   // few rows: a wave waits for memory once
  else if (pieces <= 512) SA_STREAMS(256, 2);
  else SA_STREAMS(256, 4);
#undef SA_STREAMS
}

}  // namespace sa

using namespace sa;

extern "C" int sa_streams(const float* x, int64_t x_row, int64_t x_stream, float* h, int S, const void* y, int y_dtype,
                          int64_t y_stride, int planes, const float* mix, const float* out_w, const float* in_w,
                          const void* w, int w_dtype, float eps, const int* rows, void* out, int out_dtype, int T, int D,
                          hipStream_t stream) {
  if (T == 0) return 0;
  SA_REQUIRE(T > 0 && D > 0 && D <= 16384 && S >= 1 && S <= kMaxStreams, "streams: bad sizes T=%d D=%d S=%d (at most 16384, %d)",
             T, D, S, kMaxStreams);
  SA_REQUIRE(x != nullptr && x_row >= D && x_stream >= 0, "streams: a null pointer or rows that are too short");
  SA_REQUIRE(y == nullptr || (h != nullptr && mix != nullptr && out_w != nullptr && rows == nullptr),
             "streams: an update has streams to write and its weights, and takes all rows");
  SA_REQUIRE(planes >= 0 && (planes == 0 || (y != nullptr && out_dtype == kBF16)), "streams: partial sums belong to bfloat16");
  SA_REQUIRE(in_w == nullptr || out != nullptr, "streams: nowhere to put what is read");
  SA_REQUIRE(y != nullptr || in_w != nullptr, "streams: nothing to do");
  SA_REQUIRE((out_dtype == kF32 || out_dtype == kBF16) && (w == nullptr || w_dtype == kF32 || w_dtype == kBF16) &&
                 (y == nullptr || planes > 0 || y_dtype == out_dtype),
             "streams: y and what is read have the activation type");
  Streams p;
  p.x_row = x_row, p.x_stream = x_stream, p.y_stride = y_stride, p.S = S, p.planes = planes, p.T = T, p.D = D, p.eps = eps;
  auto aligned = [](const void* q, int n) { return reinterpret_cast<uintptr_t>(q) % n == 0; };
  const bool pieces = (S == 2 || S == 4) && D % 4 == 0 && D <= 8192 && x_row % 4 == 0 && x_stream % 4 == 0 && y_stride % 4 == 0 &&
                      aligned(x, 16) && aligned(h, 16) && aligned(y, 16) && aligned(out, 16);
  if (!pieces) {
    const size_t smem = in_w != nullptr ? sizeof(float) * D : 0;
    streams_any_kernel<<<T, 256, smem, stream>>>(x, p, h, y, y_dtype, mix, out_w, in_w, w, w_dtype, rows, out, out_dtype);
    return check_launch("streams");
  }
#define SA_STREAMS_S(T_, W_)                                                                                        \
  do {                                                                                                              \
    if (S == 2) launch_streams<T_, W_, 2>(x, p, h, y, mix, out_w, in_w, w, rows, out, stream);                        \
    else launch_streams<T_, W_, 4>(x, p, h, y, mix, out_w, in_w, w, rows, out, stream);                               \
  } while (0)
  if (out_dtype == kBF16) {
    if (w_dtype == kBF16) SA_STREAMS_S(bf16, bf16);
    else SA_STREAMS_S(bf16, float);
  } else {
    if (w_dtype == kBF16) SA_STREAMS_S(float, bf16);
    else SA_STREAMS_S(float, float);
  }
#undef SA_STREAMS_S
  return check_launch("streams");
}
