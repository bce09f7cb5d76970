// The recurrence of linear_state.hip with one decay and one input factor per head, for portions of prompts, on the matrix
// cores: tokens are taken 64 at a time.  With L_t the sum of the decays' logarithms up to token t of such a piece, c_t the
// input factors and S the state in front of it,
//
//   o_i = exp(L_i) S^T q_i + sum_(j <= i) (q_i . k_j) exp(L_i - L_j) c_j v_j  (+ skip v_i)
//   S  <- exp(L_64) S + sum_j exp(L_64 - L_j) c_j k_j v_j^T
//
// A workgroup of four waves takes 16 value columns of one head of one request and walks through the pieces; the state of
// its columns stays in registers (a wave holds a quarter of the key channels) and, for reading, in LDS.  Wave w computes
// the results of tokens 16 w .. 16 w + 15.  Products with the state, with the weights exp(L_i - L_j) c_j and of the
// update are 32-bit matrix instructions (v_mfma_f32_16x16x4_f32), so the state and everything that enters it besides q, k
// and v stays 32-bit; q . k of bfloat16 rows is v_mfma_f32_16x16x32_bf16 (exact products, 32-bit sums).
//
// Everything is laid out so that a result is the next operand as it lies in registers.  A 16 x 16 result holds rows
// 4 g + r (g = lane / 16, r = 0 .. 3) and column lane % 16; an operand of k-step r holds k = g.  A sum over k may run in any
// order, so step r takes k = 4 g + r of both operands: what a lane needs of a row of q or k for the four steps is four
// neighbouring entries.  The transposed products (weights as [key token, query token], results as [value column, query
// token]) then need no exchange between lanes.
#include "api.h"
#include "attention_common.h"

namespace sa {

constexpr int kPieceTokens = 64;

struct StateChunks {
  int64_t proj_stride, gates_stride, state_stride;
  int q_at, k_at, v_at, H, heads_per_key, dk, dv, skip_dtype;
};

// An entry's bits in a 32-bit register, and its value.
__device__ __forceinline__ unsigned load_bits(const bf16* p) { return p->bits; }
__device__ __forceinline__ unsigned load_bits(const float* p) { return __float_as_uint(*p); }
template <typename XT>
__device__ __forceinline__ float bits_float(unsigned v) {
  return __uint_as_float(sizeof(XT) == 2 ? v << 16 : v);
}

// A run whose products have bfloat16 operands takes the hardware's exponential, a 32-bit run the library's.
template <bool HALF>
__device__ __forceinline__ float decay_exp(float x) {
  if constexpr (HALF) return __expf(x);
  else return expf(x);
}

// What a piece's tokens weigh, one entry per token.
struct Piece {
  double cum[kPieceTokens];                              // L_j
  __attribute__((aligned(16))) float in[kPieceTokens];   // c_j
  __attribute__((aligned(16))) float to_block[kPieceTokens];   // exp(L at the end of the token's 16 - L_j) c_j
  __attribute__((aligned(16))) float to_end[kPieceTokens];     // exp(L at the piece's end - L_j) c_j
};

// By one wave: lane j has token j's logarithm and input factor.  The sums are 64-bit, so that the differences of sums of up
// to 64 logarithms keep 32 bits.
template <bool HALF>
__device__ inline void weigh_piece(Piece& out, double lg, float in, int lane) {
  double cum = lg;
#pragma unroll
  for (int by = 1; by < kWave; by *= 2) {
    const double up = __shfl_up(cum, by, kWave);
    if (lane >= by) cum += up;
  }
  const double block = __shfl(cum, lane | 15, kWave), end = __shfl(cum, kWave - 1, kWave);
  out.cum[lane] = cum;
  out.in[lane] = in;
  out.to_block[lane] = decay_exp<HALF>(static_cast<float>(block - cum)) * in;
  out.to_end[lane] = decay_exp<HALF>(static_cast<float>(end - cum)) * in;
}

// NT: blocks of 16 key channels (dk <= 16 NT), a multiple of four.
template <int NT, typename XT>
__global__ __launch_bounds__(256) void state_chunks_kernel(const XT* __restrict__ proj, StateChunks p,
                                                           const float* __restrict__ gates, const void* __restrict__ skip,
                                                           float* __restrict__ state, const int* __restrict__ seq_meta,
                                                           float* __restrict__ out) {
  constexpr bool HALF = sizeof(XT) == 2;
  constexpr int NW = NT / 4;                     // blocks of key channels whose state a wave holds
  constexpr int ROW = NT * 16 + (HALF ? 8 : 4);  // entries of a row of k in LDS
  constexpr int VEC = HALF ? 8 : 4;              // entries of a 16-byte piece
  constexpr int PIECES = NT * 16 / VEC;          // of a row
  constexpr int PB = kPieceTokens * PIECES / 256;
  __shared__ __align__(16) XT k_s[kPieceTokens * ROW];
  __shared__ __align__(16) floatx4 s_s[2][NT * kWave];   // the state as the operand of the products that read it
  __shared__ Piece piece_s[2];
  const int* meta = seq_meta + 4 * blockIdx.x;
  const int slot = meta[0], first = meta[1], count = meta[2];
  if (count <= 0) return;
  const int h = blockIdx.y, tid = threadIdx.x, lane = tid % kWave;
  const int wave = __builtin_amdgcn_readfirstlane(tid / kWave);
  const int c = lane % 16, g = lane / 16;
  const int kh = h / p.heads_per_key;
  const int col = blockIdx.z * 16 + c;
  const bool col_ok = col < p.dv;
  float* S = state + static_cast<size_t>(slot) * p.state_stride + static_cast<size_t>(h) * p.dk * p.dv;

  // the wave's part of the state: key channels 16 (wave NW + n) + 4 g + r of value column c
  floatx4 s[NW];
#pragma unroll
  for (int n = 0; n < NW; ++n) {
    const int d = (wave * NW + n) * 16 + g * 4;
    s[n] = floatx4{0.f, 0.f, 0.f, 0.f};
    if (col_ok && d < p.dk) s[n] = *reinterpret_cast<const floatx4*>(S + static_cast<size_t>(col) * p.dk + d);
    s_s[0][(wave * NW + n) * kWave + lane] = s[n];
  }
  float sk = 0.f;
  if (skip != nullptr) sk = load_f(skip, p.skip_dtype, h);

  // what a piece needs from memory, asked for a piece ahead
  uint4 kb[PB];                    // rows of k, on their way to LDS
  unsigned vb[16];                 // the bits of v[16 b + 4 g + r][c]
  uint4 qb[HALF ? NT / 2 : NT];    // four neighbouring entries of the wave's own rows of q per block of key channels
  unsigned xb[4];                  // and of v of the lane's own token, four columns, for the skip
  float lg = 0.f, in = 0.f;        // a token a lane: the decay's logarithm and the input factor
  const int own = wave * 16 + c;   // the lane's own token of the piece
  // A lane's places in a piece: 32-bit offsets from rows that are the same for all lanes, without a branch, so that nothing
  // waits for the loads before they are used.  (tokens behind the request's last one stand for the last one again: their
  // input factor is 0, their results go nowhere; channels behind the last meet zeros in k and in the state)
  const int stride = static_cast<int>(p.proj_stride);
  const int k_lane = tid / PIECES, k_d = tid % PIECES * VEC;   // (256 threads: whole rows of k each time)
  const int k_col = k_d < p.dk ? k_d : 0, v_col = col_ok ? col : 0;
  const int x_col = blockIdx.z * 16 + g * 4 < p.dv ? blockIdx.z * 16 + g * 4 : 0;   // (value sizes are multiples of 4)
  auto fetch = [&](int t0) __attribute__((always_inline)) {
    const int last = (count - t0 < kPieceTokens ? count - t0 : kPieceTokens) - 1;
    const XT* rows = proj + static_cast<size_t>(first + t0) * p.proj_stride;
    auto row = [&](int j) __attribute__((always_inline)) { return (j < last ? j : last) * stride; };
    const XT* kp = rows + p.k_at + kh * p.dk;
    const XT* vp = rows + p.v_at + h * p.dv;
    const XT* qp = rows + p.q_at + kh * p.dk;
#pragma unroll
    for (int i = 0; i < PB; ++i) kb[i] = *reinterpret_cast<const uint4*>(kp + row(k_lane + i * (256 / PIECES)) + k_col);
#pragma unroll
    for (int i = 0; i < 16; ++i) vb[i] = load_bits(vp + row(i / 4 * 16 + g * 4 + i % 4) + v_col);
    const int mine = row(own);
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const int d = n * 16 + g * 4, at = mine + (d < p.dk ? d : 0);
      if constexpr (HALF) {
        const uint2 v = *reinterpret_cast<const uint2*>(qp + at);
        if (n % 2 == 0) qb[n / 2].x = v.x, qb[n / 2].y = v.y;
        else qb[n / 2].z = v.x, qb[n / 2].w = v.y;
      } else {
        qb[n] = *reinterpret_cast<const uint4*>(qp + at);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) xb[r] = load_bits(vp + mine + x_col + r);
    const float* gr = gates + static_cast<size_t>(first + t0 + (lane < last ? lane : last)) * p.gates_stride;
    in = gr[p.H + h];
    lg = gr[2 * p.H + h];
  };
  auto weigh = [&](Piece& to, int t0) __attribute__((always_inline)) {
    const bool live = t0 + lane < count;
    weigh_piece<HALF>(to, live ? lg : 0.f, live ? in : 0.f, lane);
  };
  fetch(0);
  if (wave == 0) weigh(piece_s[0], 0);
  int now = 0;
  for (int t0 = 0; t0 < count; t0 += kPieceTokens, now ^= 1) {
    __syncthreads();   // (the piece before has been worked through)
#pragma unroll
    for (int i = 0; i < PB; ++i) {
      const int idx = tid + i * 256;
      *reinterpret_cast<uint4*>(&k_s[idx / PIECES * ROW + idx % PIECES * VEC]) = idx % PIECES * VEC < p.dk ? kb[i] : uint4{0, 0, 0, 0};
    }
    float v[16], x[4];
#pragma unroll
    for (int i = 0; i < 16; ++i) v[i] = bits_float<XT>(vb[i]);
#pragma unroll
    for (int r = 0; r < 4; ++r) x[r] = bits_float<XT>(xb[r]);
    uint4 q[HALF ? NT / 2 : NT];
#pragma unroll
    for (int n = 0; n < (HALF ? NT / 2 : NT); ++n) q[n] = qb[n];
    __syncthreads();
    fetch(t0 + kPieceTokens < count ? t0 + kPieceTokens : t0);   // (behind the last piece: that one again, for nothing)

    // o^T[column, own token] from the state
    floatx4 o{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const floatx4 st = s_s[now][n * kWave + lane];
      floatx4 qf;
      if constexpr (HALF) {
        const unsigned lo = n % 2 == 0 ? q[n / 2].x : q[n / 2].z, hi = n % 2 == 0 ? q[n / 2].y : q[n / 2].w;
        qf = floatx4{__uint_as_float(lo << 16), __uint_as_float(lo & 0xffff0000u), __uint_as_float(hi << 16),
                     __uint_as_float(hi & 0xffff0000u)};
      } else {
        qf = __builtin_bit_cast(floatx4, q[n]);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) o = __builtin_amdgcn_mfma_f32_16x16x4f32(st[r], qf[r], o, 0, 0, 0);
    }
    const Piece& pc = piece_s[now];
    const double cum_i = pc.cum[own];
    {
      const float e = decay_exp<HALF>(static_cast<float>(cum_i));
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] *= e;
    }
    // and from the piece's own tokens, 16 of them at a time: weights [token j, own token], exp(L_i - L_j) c_j: in an
    // earlier block by way of that block's end, in the own one token by token (tokens behind the own one: exp of minus
    // infinity)
    floatx4 own_wgt = *reinterpret_cast<const floatx4*>(&pc.in[wave * 16 + g * 4]);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int j = wave * 16 + g * 4 + r;
      const float d = static_cast<float>(cum_i - pc.cum[j]);
      own_wgt[r] *= decay_exp<HALF>(j <= own ? d : -INFINITY);
    }
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      if (b > wave) break;   // (uniform over the wave)
      floatx4 m{0.f, 0.f, 0.f, 0.f};
      const XT* kr = &k_s[(b * 16 + c) * ROW + g * 4];
      if constexpr (HALF) {
#pragma unroll
        for (int n = 0; n < NT / 2; ++n) {
          const uint2 lo = *reinterpret_cast<const uint2*>(kr + n * 32), hi = *reinterpret_cast<const uint2*>(kr + n * 32 + 16);
          const uint4 kk{lo.x, lo.y, hi.x, hi.y};
          m = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, kk), __builtin_bit_cast(bf16x8, q[n]), m, 0, 0, 0);
        }
      } else {
#pragma unroll
        for (int n = 0; n < NT; ++n) {
          const floatx4 kf = *reinterpret_cast<const floatx4*>(kr + n * 16), qf = __builtin_bit_cast(floatx4, q[n]);
#pragma unroll
          for (int r = 0; r < 4; ++r) m = __builtin_amdgcn_mfma_f32_16x16x4f32(kf[r], qf[r], m, 0, 0, 0);
        }
      }
      floatx4 wgt = own_wgt;
      if (b < wave) {
        const float e = decay_exp<HALF>(static_cast<float>(cum_i - pc.cum[b * 16 + 15]));
        wgt = *reinterpret_cast<const floatx4*>(&pc.to_block[b * 16 + g * 4]);
#pragma unroll
        for (int r = 0; r < 4; ++r) wgt[r] *= e;
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) o = __builtin_amdgcn_mfma_f32_16x16x4f32(v[b * 4 + r], m[r] * wgt[r], o, 0, 0, 0);
    }
    if (t0 + own < count) {
      const int cc = blockIdx.z * 16 + g * 4;
      float* dst = out + static_cast<size_t>(first + t0 + own) * (static_cast<size_t>(p.H) * p.dv) + static_cast<size_t>(h) * p.dv + cc;
      floatx4 y;
#pragma unroll
      for (int r = 0; r < 4; ++r) y[r] = fmaf(sk, x[r], o[r]);
      if (cc < p.dv) *reinterpret_cast<floatx4*>(dst) = y;
    }
    // the state behind the piece
    const float all = decay_exp<HALF>(static_cast<float>(pc.cum[kPieceTokens - 1]));
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      const floatx4 e = *reinterpret_cast<const floatx4*>(&pc.to_end[b * 16 + g * 4]);
#pragma unroll
      for (int r = 0; r < 4; ++r) v[b * 4 + r] *= e[r];
    }
#pragma unroll
    for (int n = 0; n < NW; ++n) {
      const int nb = wave * NW + n;
#pragma unroll
      for (int r = 0; r < 4; ++r) s[n][r] *= all;
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int j = i / 4 * 16 + g * 4 + i % 4;
        s[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(to_float(k_s[j * ROW + nb * 16 + c]), v[i], s[n], 0, 0, 0);
      }
      s_s[now ^ 1][nb * kWave + lane] = s[n];
    }
    // (by the wave with the fewest blocks of tokens to go through)
    if (wave == 0 && t0 + kPieceTokens < count) weigh(piece_s[now ^ 1], t0 + kPieceTokens);
  }
#pragma unroll
  for (int n = 0; n < NW; ++n) {
    const int d = (wave * NW + n) * 16 + g * 4;
    if (col_ok && d < p.dk) *reinterpret_cast<floatx4*>(S + static_cast<size_t>(col) * p.dk + d) = s[n];
  }
}

}  // namespace sa

using namespace sa;

extern "C" int sa_state_chunks_takes(int dk, int dv, int q_at, int k_at, int v_at, int64_t proj_stride, int64_t state_stride) {
  return dk > 0 && dk <= 128 && dk % 8 == 0 && dv > 0 && dv % 4 == 0 && q_at % 8 == 0 && k_at % 8 == 0 && v_at >= 0 &&
         proj_stride % 8 == 0 && state_stride % 4 == 0;
}

extern "C" int sa_state_chunks(const void* proj, int dtype, int64_t proj_stride, int q_at, int k_at, int v_at,
                               const float* gates, int64_t gates_stride, const void* skip, int skip_dtype, int H, int key_heads,
                               int dk, int dv, float* state, int64_t state_stride, const int* seq_meta, int num_seqs, float* out,
                               hipStream_t stream) {
  if (num_seqs == 0) return 0;
  SA_REQUIRE(num_seqs > 0 && H > 0 && H <= 65535 && key_heads > 0 && H % key_heads == 0, "state_chunks: bad sizes S=%d H=%d", num_seqs, H);
  SA_REQUIRE(sa_state_chunks_takes(dk, dv, q_at, k_at, v_at, proj_stride, state_stride),
             "state_chunks: does not take keys of %d and values of %d at columns %d, %d", dk, dv, q_at, k_at);
  SA_REQUIRE(proj != nullptr && gates != nullptr && state != nullptr && seq_meta != nullptr && out != nullptr &&
                 reinterpret_cast<uintptr_t>(proj) % 16 == 0 && reinterpret_cast<uintptr_t>(state) % 16 == 0 &&
                 reinterpret_cast<uintptr_t>(out) % 16 == 0,
             "state_chunks: a null or unaligned pointer");
  SA_REQUIRE(state_stride >= static_cast<int64_t>(H) * dk * dv && gates_stride >= 3 * H && q_at >= 0 && k_at >= 0 &&
                 proj_stride >= q_at + static_cast<int64_t>(key_heads) * dk && proj_stride >= k_at + static_cast<int64_t>(key_heads) * dk &&
                 proj_stride >= v_at + static_cast<int64_t>(H) * dv,
             "state_chunks: rows of the state, the gates or the projection are too short");
  SA_REQUIRE(proj_stride * kPieceTokens < (1LL << 31), "state_chunks: rows of %lld entries are too long", (long long)proj_stride);
  SA_REQUIRE((dtype == kF32 || dtype == kBF16) && (skip == nullptr || skip_dtype == kF32 || skip_dtype == kBF16),
             "state_chunks: unknown dtype");
  StateChunks p;
  p.proj_stride = proj_stride, p.gates_stride = gates_stride, p.state_stride = state_stride, p.q_at = q_at, p.k_at = k_at;
  p.v_at = v_at, p.H = H, p.heads_per_key = H / key_heads, p.dk = dk, p.dv = dv, p.skip_dtype = skip_dtype;
  const dim3 grid(num_seqs, H, (dv + 15) / 16);
#define SA_CHUNKS(NT, XT) \
  state_chunks_kernel<NT, XT><<<grid, 256, 0, stream>>>(static_cast<const XT*>(proj), p, gates, skip, state, seq_meta, out)
  if (dtype == kBF16) {
    if (dk <= 64) SA_CHUNKS(4, bf16);
    else SA_CHUNKS(8, bf16);
  } else {
    if (dk <= 64) SA_CHUNKS(4, float);
    else SA_CHUNKS(8, float);
  }
#undef SA_CHUNKS
  return check_launch("state_chunks");
}
