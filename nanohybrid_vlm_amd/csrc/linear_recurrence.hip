// Linear recurrences: mixers whose state is one matrix S[D, E] per head and request that decays and takes one outer
// product a token, without a softmax or a denominator. Two designs of them share the kernels (kind):
//   kind 0, a fixed decay per head ("retention"):      S_t = g_h S_(t-1) + k_t v_t^T,           o_t = S_t^T q_t,
//           q and k turned by position (pairs (i, i + rot / 2)), k multiplied by a constant;
//   kind 1, a decay per key channel and token ("wkv"): o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t, S_t = diag(w_t) S_(t-1) + k_t v_t^T,
//           w = exp(-exp(W2 tanh(z) + w0)) with z the first product of a low-rank projection.
// Kernels:
//  - nhv_token_shift: rows mixed with the row before them, x + (x' - x) mu_i, for several mu at once; the row before a
//    request's first row of the step is kept per request;
//  - nhv_recurrence_prepare and nhv_recurrence_chunks: portions of prompts, 16 tokens at a time. The first works on all
//    chunks at once: decays and their running products, the products of a chunk's tokens among themselves
//    A[t, j] (j <= t), queries with the decay from the chunk's start R[t], keys with the decay to its end K[t], and
//    the decay of the whole chunk. The second walks over a request's chunks in order: O = A V + R S, S = diag(decay) S + K^T V,
//    as float matrix products (v_mfma_f32_16x16x4_f32);
//  - nhv_recurrence_tokens: steps of one or a few tokens a request: everything from the projections to the normed and
//    gated read-out in one launch, a block per (request, head);
//  - nhv_readout_norm: o over its root mean square per head, times a weight per entry (optional), times g sigmoid(g).
// Everything is float but the projections' rows. Decays are kept as base-2 logarithms and only differences that are
// never positive are raised: a strong decay gives zeros, not overflows. The state is [slots, H, E, D], zero for a request whose
// first token is at position 0. A request without tokens in the step is left alone. A token's sums within a step
// depend on where the step's first token of its request lies, by rounding only.
#include "nhv_common.h"
#include "nhv_rotation.h"
#include <math.h>

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;

#define NHV_LOG2E 1.4426950408889634f
#define NHV_CHUNK 16

__device__ __forceinline__ float exp2_of(float x) { return __builtin_amdgcn_exp2f(x); }   // (x <= 0; tiny results may become 0)
__device__ __forceinline__ float silu_of(float z) { return z / (1.0f + expf(-z)); }

// ---------------------------------------------------------------- rows mixed with the row before them
// out[i, t, :] = h[t] + (h' - h[t]) mu[i], h' the request's row before t (of this step, or kept[slot]; zeros at position 0).
// The thread that reads a kept row (the request's first row of the step) also writes what the next step needs: the
// request's last row; no other thread touches the kept row.
template <typename T, int V>
__global__ __launch_bounds__(256) void token_shift_kernel(const T* __restrict__ h, const float* __restrict__ mu, float* kept,
                                                          T* __restrict__ out, const int* __restrict__ token_req,
                                                          const int* __restrict__ positions, const int* __restrict__ cu,
                                                          const int* __restrict__ state_slots, int n_mu, int rows, int W) {
  struct alignas(sizeof(T) * V) Pack { T e[V]; };
  const int c = (blockIdx.x * 256 + threadIdx.x) * V;
  if (c >= W) return;
  for (int t = blockIdx.y; t < rows; t += gridDim.y) {
    const int req = token_req[t], first = cu[req];
    const Pack me = *reinterpret_cast<const Pack*>(h + (size_t)t * W + c);
    float x[V], d[V];
    if (t > first) {
      const Pack before = *reinterpret_cast<const Pack*>(h + (size_t)(t - 1) * W + c);
#pragma unroll
      for (int i = 0; i < V; ++i) d[i] = to_f32(before.e[i]);
    } else {
      float* row = kept + (size_t)state_slots[req] * W + c;
      const bool fresh = positions[t] == 0;
#pragma unroll
      for (int i = 0; i < V; ++i) d[i] = fresh ? 0.f : row[i];
      const Pack last = *reinterpret_cast<const Pack*>(h + (size_t)(cu[req + 1] - 1) * W + c);
#pragma unroll
      for (int i = 0; i < V; ++i) row[i] = to_f32(last.e[i]);
    }
#pragma unroll
    for (int i = 0; i < V; ++i) {
      x[i] = to_f32(me.e[i]);
      d[i] -= x[i];
    }
    for (int m = 0; m < n_mu; ++m) {
      Pack y;
#pragma unroll
      for (int i = 0; i < V; ++i) y.e[i] = from_f32<T>(fmaf(d[i], mu[(size_t)m * W + c + i], x[i]));
      *reinterpret_cast<Pack*>(out + ((size_t)m * rows + t) * W + c) = y;
    }
  }
}

extern "C" int nhv_token_shift(const void* h, const void* mu, void* kept, void* out, const void* token_req, const void* positions,
                               const void* cu, const void* state_slots, int n_mu, int T, int W, int dtype, void* stream) {
  NHV_REQUIRE(T > 0 && W > 0 && n_mu > 0, "token_shift: bad sizes T=%d W=%d mixes=%d", T, W, n_mu);
  hipStream_t s = (hipStream_t)stream;
  const bool wide = W % 8 == 0 && (((uintptr_t)h | (uintptr_t)out) & 31) == 0;
#define LAUNCH(TT, VV)                                                                                                  \
  hipLaunchKernelGGL((token_shift_kernel<TT, VV>), dim3((W / VV + 255) / 256, T < 65535 ? T : 65535), dim3(256), 0, s,   \
                     (const TT*)h, (const float*)mu, (float*)kept, (TT*)out, (const int*)token_req, (const int*)positions, \
                     (const int*)cu, (const int*)state_slots, n_mu, T, W)
  if (dtype == NHV_F32) { if (wide) LAUNCH(float, 8); else LAUNCH(float, 1); }
  else if (dtype == NHV_BF16) { if (wide) LAUNCH(bf16_t, 8); else LAUNCH(bf16_t, 1); }
  else return nhv_fail("token_shift: unknown dtype %d", dtype);
#undef LAUNCH
  NHV_LAUNCH_CHECK("token_shift");
  return 0;
}

// ---------------------------------------------------------------- what the recurrences read
// Rows of q (or r), k, v and the gates' linear parts: entry (t, h, i) at ptr + t ld + h size + i, all of one type.
struct RecurrenceIn {
  const void* q;
  const void* k;
  const void* v;
  const void* g;
  long long ld;
  // kind 0
  const float* log2_decay;                   // [H]
  const double* freqs;                       // [rot / 2]
  const int* turn_positions;                 // [T]
  int rot;
  float k_scale;
  // kind 1
  const float* z;                            // [T, rank], rows z_ld apart: before the tanh
  long long z_ld;
  const void* w2;                            // [H D, rank] of the weights' type
  int rank;
  const float* w0;                           // [H D]
  const float* u;                            // [H D]
};


// four consecutive entries (``whole``: they start at a multiple of four, else one by one, those from n on being zeros)
template <typename T>
__device__ __forceinline__ floatx4 four_of(const T* p, int n, bool whole) {
  struct alignas(sizeof(T) * 4) Pack { T e[4]; };
  floatx4 v;
  if (whole) {
    const Pack x = *reinterpret_cast<const Pack*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = to_f32(x.e[i]);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = i < n ? to_f32(p[i]) : 0.f;
  }
  return v;
}

// ---------------------------------------------------------------- portions of prompts: all chunks at once
// One block of 256 threads per (chunk, head, request). A chunk's place in the outputs: cu[req] / 16 + req + its number in
// the request (places never overlap: a request of n tokens has at most floor(n / 16) + 1 chunks). ``whole``: rows, heads and
// ranks are whole groups of four entries.
template <typename T, typename TW, int KIND>
__global__ __launch_bounds__(256) void recurrence_prepare_kernel(const RecurrenceIn in, float* __restrict__ r_out,
                                                                 float* __restrict__ k_out, float* __restrict__ a_out,
                                                                 float* __restrict__ decay_out, const int* __restrict__ cu,
                                                                 int H, int D, int Dp, int whole, int whole_rank) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int req = blockIdx.z, h = blockIdx.x;
  const int first = cu[req], t0 = first + blockIdx.y * NHV_CHUNK, end = cu[req + 1];
  if (t0 >= end) return;                     // (the same for the whole block)
  const int n = min(NHV_CHUNK, end - t0);
  const size_t place = ((size_t)(first / NHV_CHUNK) + req + blockIdx.y) * H + h;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, col = lane & 15, grp = lane >> 4;
  const int LD = Dp + 4;                     // (an odd number of groups of four: sixteen rows' groups lie in sixty-four banks)
  float* rs = lds;
  float* ks = rs + NHV_CHUNK * LD;
  float* ls = ks + NHV_CHUNK * LD;           // kind 1: running sums of the decays' logarithms, the token's own included
  const T* q = (const T*)in.q + (size_t)h * D;
  const T* k = (const T*)in.k + (size_t)h * D;
  const floatx4 zero = {0.f, 0.f, 0.f, 0.f};
  const int fours = Dp / 4;
  if (KIND == 1) {
    // the decays' linear part tanh(z) w2^T on the matrix cores: a wave takes every fourth tile of 16 channels
    constexpr int MAX_TILES = 4;
    floatx4 acc[MAX_TILES];
#pragma unroll
    for (int i = 0; i < MAX_TILES; ++i) acc[i] = zero;
    const float* z = in.z + (size_t)(t0 + min(col, n - 1)) * in.z_ld;
    for (int r0 = 0; r0 < in.rank; r0 += 16) {
      const int r = r0 + grp * 4;
      floatx4 x, w[MAX_TILES];
#pragma unroll
      for (int j = 0; j < 4; ++j) x[j] = r + j < in.rank ? z[r + j] : 0.f;
#pragma unroll
      for (int i = 0; i < MAX_TILES; ++i) {
        const int d = (wave + 4 * i) * 16 + col;
        w[i] = (d < D && r < in.rank) ? four_of((const TW*)in.w2 + ((size_t)h * D + d) * in.rank + r, in.rank - r, whole_rank) : zero;
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) x[j] = tanhf(x[j]);
#pragma unroll
      for (int i = 0; i < MAX_TILES; ++i)
        if ((wave + 4 * i) * 16 < Dp)
#pragma unroll
          for (int j = 0; j < 4; ++j) acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(x[j], w[i][j], acc[i], 0, 0, 0);
    }
    // a lane holds channel d at the tokens 4 grp .. 4 grp + 3: sums along them, then over the groups before
#pragma unroll
    for (int i = 0; i < MAX_TILES; ++i) {
      const int d = (wave + 4 * i) * 16 + col;
      if (d - col >= Dp) continue;           // (the same for the whole wave)
      const float w0 = d < D ? in.w0[h * D + d] : 0.f;
      float run[4], sum = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const bool real = d < D && grp * 4 + j < n;
        sum += real ? -NHV_LOG2E * expf(acc[i][j] + w0) : 0.f;
        run[j] = sum;
      }
      const float s0 = __shfl(sum, col, NHV_WAVE), s1 = __shfl(sum, col + 16, NHV_WAVE), s2 = __shfl(sum, col + 32, NHV_WAVE);
      const float before = grp == 0 ? 0.f : grp == 1 ? s0 : grp == 2 ? s0 + s1 : s0 + s1 + s2;
#pragma unroll
      for (int j = 0; j < 4; ++j) ls[(grp * 4 + j) * LD + d] = before + run[j];
    }
  }
  const int half = KIND == 0 ? in.rot / 2 : 0;
  if (KIND == 0 && half > 0) {
    const bool fast = whole && half % 4 == 0;
    for (int x = tid; x < NHV_CHUNK * (fast ? half / 4 : half); x += 256) {
      const int per = fast ? half / 4 : half;
      const int t = x / per, i = (x % per) * (fast ? 4 : 1);
      const size_t at = (size_t)(t0 + t) * in.ld + i;
      floatx4 q1 = zero, q2 = zero, k1 = zero, k2 = zero;
      if (t < n) {
        const int count = fast ? 4 : 1;
        q1 = four_of(q + at, count, fast); q2 = four_of(q + at + half, count, fast);
        k1 = four_of(k + at, count, fast); k2 = four_of(k + at + half, count, fast);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        if (j > 0 && !fast) break;
        float sn = 0.f, cs = 1.f;
        if (t < n) nhv_turn_angle<float>(in.turn_positions[t0 + t], in.freqs[i + j], 1.0f, &sn, &cs);
        rs[t * LD + i + j] = q1[j] * cs - q2[j] * sn;
        rs[t * LD + i + j + half] = q2[j] * cs + q1[j] * sn;
        ks[t * LD + i + j] = (k1[j] * cs - k2[j] * sn) * in.k_scale;
        ks[t * LD + i + j + half] = (k2[j] * cs + k1[j] * sn) * in.k_scale;
      }
    }
  }
  {                                          // what is not turned, and the places beyond D
    const float k_scale = KIND == 0 ? in.k_scale : 1.0f;
    const int start = 2 * half, f0 = start / 4;
    const bool fast = whole && start % 4 == 0;
    for (int x = tid; x < NHV_CHUNK * (fours - f0); x += 256) {
      const int t = x / (fours - f0), d = (x % (fours - f0) + f0) * 4;
      const size_t at = (size_t)(t0 + t) * in.ld + d;
      if (fast) {
        const bool real = t < n && d < D;
        *reinterpret_cast<floatx4*>(&rs[t * LD + d]) = real ? four_of(q + at, 4, true) : zero;
        floatx4 kv = real ? four_of(k + at, 4, true) : zero;
        kv *= k_scale;
        *reinterpret_cast<floatx4*>(&ks[t * LD + d]) = kv;
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          if (d + j < start) continue;
          const bool real = t < n && d + j < D;
          rs[t * LD + d + j] = real ? to_f32(q[at + j]) : 0.f;
          ks[t * LD + d + j] = real ? to_f32(k[at + j]) * k_scale : 0.f;
        }
      }
    }
  }
  __syncthreads();
  const float l2 = KIND == 0 ? in.log2_decay[h] : 0.f;
  {                                          // A: a thread per (t, j)
    const int t = tid >> 4, j = tid & 15;
    float sum = 0.f;
    if (t < n && j <= t) {
      const float* rt = rs + t * LD;
      const float* kj = ks + j * LD;
      floatx4 part = zero;
      if (KIND == 0) {
        for (int d = 0; d < Dp; d += 4) part += *reinterpret_cast<const floatx4*>(rt + d) * *reinterpret_cast<const floatx4*>(kj + d);
        sum = (part[0] + part[1] + part[2] + part[3]) * exp2_of(l2 * (float)(t - j));
      } else if (j == t) {
        for (int d = 0; d < D; ++d) sum = fmaf(rt[d] * in.u[h * D + d], kj[d], sum);
      } else {
        const float* lt = ls + (t - 1) * LD;
        const float* lj = ls + j * LD;
#pragma unroll 2
        for (int d = 0; d < Dp; d += 4) {
          const floatx4 x = *reinterpret_cast<const floatx4*>(lt + d) - *reinterpret_cast<const floatx4*>(lj + d);
          floatx4 e;
#pragma unroll
          for (int i = 0; i < 4; ++i) e[i] = exp2_of(x[i]);
          part += *reinterpret_cast<const floatx4*>(rt + d) * *reinterpret_cast<const floatx4*>(kj + d) * e;
        }
        sum = part[0] + part[1] + part[2] + part[3];
      }
    }
    a_out[place * 256 + tid] = sum;
  }
  for (int x = tid; x < NHV_CHUNK * fours; x += 256) {
    const int t = x / fours, d = (x % fours) * 4;
    floatx4 r = *reinterpret_cast<const floatx4*>(&rs[t * LD + d]);
    if (KIND == 0) {
      r *= exp2_of(l2 * (float)(t + 1));
    } else if (t > 0) {
      const floatx4 before = *reinterpret_cast<const floatx4*>(&ls[(t - 1) * LD + d]);
#pragma unroll
      for (int j = 0; j < 4; ++j) r[j] *= exp2_of(before[j]);
    }
    *reinterpret_cast<floatx4*>(r_out + place * NHV_CHUNK * Dp + x * 4) = r;
  }
  for (int x = tid; x < Dp * 4; x += 256) {  // keys lie with a channel's sixteen tokens together
    const int t = (x & 3) * 4, d = x >> 2;
    floatx4 kk;
#pragma unroll
    for (int j = 0; j < 4; ++j)              // (rows beyond n are zeros)
      kk[j] = ks[(t + j) * LD + d] * exp2_of(KIND == 0 ? l2 * (float)max(n - 1 - t - j, 0) : ls[(n - 1) * LD + d] - ls[(t + j) * LD + d]);
    *reinterpret_cast<floatx4*>(k_out + place * NHV_CHUNK * Dp + x * 4) = kk;
  }
  for (int d = tid; d < Dp; d += 256)
    decay_out[place * Dp + d] = d < D ? exp2_of(KIND == 0 ? l2 * (float)n : ls[(n - 1) * LD + d]) : 0.f;
}

// ---------------------------------------------------------------- portions of prompts: a request's chunks in order
// A block owns 16 columns of S (value channels) of one head of one request; its four waves share D in tiles of 16 rows,
// TPW tiles a wave, which stay in registers as the result of the matrix cores' products: lane l holds S[16 tile + 4 (l / 16) + i,
// column l % 16]. With the rows of D taken in that same order the tile is also the right-hand operand of R S as it stands.
// The waves' shares of O meet in LDS (two buffers, one barrier a chunk) and are added in the order of the waves. What a
// chunk needs is asked for AHEAD chunks before it is used. EVEN: every wave has TPW tiles. Blocks of one head are a multiple of the number of heads
// apart, so that with a multiple of eight heads they share an XCD's L2.
template <typename T, int TPW>
struct ChunkOperands {
  floatx4 r[TPW], g[TPW], kk[TPW];
  T v[4], v_mine;
  float a;
};

// (two waves a SIMD at least: with at most 256 registers a wave the products' sums stay in ordinary registers)
template <typename T, int TPW, bool EVEN>
__global__ __launch_bounds__(256, 2) void recurrence_chunks_kernel(const float* __restrict__ r_in, const float* __restrict__ k_in,
                                                                const float* __restrict__ a_in, const float* __restrict__ decay_in,
                                                                const T* __restrict__ v, long long ld, float* __restrict__ state,
                                                                float* __restrict__ out, const int* __restrict__ positions,
                                                                const int* __restrict__ cu, const int* __restrict__ state_slots,
                                                                int H, int D, int Dp, int E) {
  constexpr int AHEAD = TPW <= 2 ? 3 : 2;
  __shared__ float red[2][4][NHV_CHUNK][17];
  const int req = blockIdx.z, h = blockIdx.x, e0 = blockIdx.y * 16;
  const int first = cu[req], end = cu[req + 1];
  if (end <= first) return;                  // (the same for the whole block)
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, col = lane & 15, grp = lane >> 4;
  const int tiles = Dp / 16, tile0 = wave * TPW;
  const bool column = e0 + col < E;
  float* mine = state + (((size_t)state_slots[req] * H + h) * E + (column ? e0 + col : 0)) * D;
  const bool fresh = positions[first] == 0;
  floatx4 S[TPW];
#pragma unroll
  for (int i = 0; i < TPW; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int d = (tile0 + i) * 16 + grp * 4 + j;
      S[i][j] = (!fresh && column && d < D) ? mine[d] : 0.f;
    }
  const int chunks = (end - first + NHV_CHUNK - 1) / NHV_CHUNK;
  const size_t place0 = (size_t)(first / NHV_CHUNK) + req;
  ChunkOperands<T, TPW> ops[AHEAD];
  // what a lane reads of a chunk lies at offsets that do not change, from bases that are the same for the whole block
  const int r_at = col * Dp + tile0 * 16 + grp * 4, k_at = (tile0 * 16 + col) * NHV_CHUNK + grp * 4, g_at = tile0 * 16 + grp * 4;
  const int a_at = col * 16 + grp * 4 + wave;
  const int spare = (EVEN ? 0 : tiles) - 1;  // (a wave without a tile reads the last one's and leaves it unused)
  const T* vbase = v + (size_t)first * ld + (size_t)h * E + e0;
  const int row = (int)ld, vlast = (end - first - 1) * row + (column ? col : 0);       // (a lane beyond E works on a column that it does not write)
  int v_at[4], v_mine_at = (grp * 4 + wave) * row + (column ? col : 0);
#pragma unroll
  for (int j = 0; j < 4; ++j) v_at[j] = (grp * 4 + j) * row + (column ? col : 0);
  auto ask = [&](ChunkOperands<T, TPW>& x, int c) {      // (in the order of the chunks)
    c = min(c, chunks - 1);                  // (always asked, so that the loop's waits count the same loads on every way)
    const size_t place = (place0 + c) * H + h;
    const float* rb = r_in + place * NHV_CHUNK * Dp;
    const float* kb = k_in + place * NHV_CHUNK * Dp;
    const float* gb = decay_in + place * Dp;
#pragma unroll
    for (int i = 0; i < TPW; ++i) {
      const int back = EVEN ? 0 : max(tile0 + i - spare, 0);
      x.r[i] = *reinterpret_cast<const floatx4*>(rb + (r_at + (i - back) * 16));
      x.g[i] = *reinterpret_cast<const floatx4*>(gb + (g_at + (i - back) * 16));
      x.kk[i] = *reinterpret_cast<const floatx4*>(kb + (k_at + (i - back) * 16 * NHV_CHUNK));
    }
    // (rows beyond the request meet zeros in A and K: the request's last row stands in for them)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      x.v[j] = vbase[min(v_at[j], vlast)];
      v_at[j] += NHV_CHUNK * row;
    }
    x.v_mine = vbase[min(v_mine_at, vlast)];
    v_mine_at += NHV_CHUNK * row;
    x.a = a_in[place * 256 + a_at];
  };
  const int o_at = (tid >> 4) * H * E + (tid & 15);
  // the waves' shares of chunk c added up and written
  auto emit = [&](int c) {
    const int t = first + c * NHV_CHUNK + (tid >> 4), e = e0 + (tid & 15);
    float sum = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) sum += red[c & 1][w][tid >> 4][tid & 15];
    float* ob = out + ((size_t)(first + c * NHV_CHUNK) * H + h) * E + e0;
    if (t < end && e < E) ob[o_at] = sum;
  };
  auto step = [&](ChunkOperands<T, TPW>& x, int c) {
    float vv[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) vv[j] = to_f32(x.v[j]);
    floatx4 o = {0.f, 0.f, 0.f, 0.f}, o2 = {0.f, 0.f, 0.f, 0.f};
    // this wave's share of A V: the tokens 4 grp + wave
    o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.a, to_f32(x.v_mine), o2, 0, 0, 0);
#pragma unroll
    for (int i = 0; i < TPW; ++i) {
      if (!EVEN && tile0 + i >= tiles) continue;      // (the same for the whole wave)
      o = __builtin_amdgcn_mfma_f32_16x16x4f32(x.r[i][0], S[i][0], o, 0, 0, 0);
      o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.r[i][1], S[i][1], o2, 0, 0, 0);
      o = __builtin_amdgcn_mfma_f32_16x16x4f32(x.r[i][2], S[i][2], o, 0, 0, 0);
      o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.r[i][3], S[i][3], o2, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < TPW; ++i) S[i] *= x.g[i];
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int i = 0; i < TPW; ++i)
        if (EVEN || tile0 + i < tiles) S[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.kk[i][j], vv[j], S[i], 0, 0, 0);
    ask(x, c + AHEAD);
    if (c > 0) emit(c - 1);                  // (while the products are under way)
#pragma unroll
    for (int j = 0; j < 4; ++j) red[c & 1][wave][grp * 4 + j][col] = o[j] + o2[j];
    // a barrier for LDS alone: __syncthreads would also wait for the loads that were asked for ahead. A buffer's sums are read
    // in the step after (below), before that step's barrier, and written again only behind it.
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
  };
#pragma unroll
  for (int i = 0; i < AHEAD; ++i) ask(ops[i], i);
  int c = 0;
  for (; c + AHEAD <= chunks; c += AHEAD) {
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) step(ops[i], c + i);
  }
#pragma unroll
  for (int i = 0; i < AHEAD - 1; ++i)
    if (c + i < chunks) step(ops[i], c + i);
  emit(chunks - 1);
#pragma unroll
  for (int i = 0; i < TPW; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int d = (tile0 + i) * 16 + grp * 4 + j;
      if (column && d < D) mine[d] = S[i][j];
    }
}

// ---------------------------------------------------------------- steps of a few tokens a request: one launch
// A block per (head, request). Token by token: the token's vectors go to LDS (turned; decays worked out), then every column
// of S meets them: a column belongs to R adjacent lanes of 16 entries each (in fours, the lanes' fours side by side: a load
// takes whole lines), columns beyond the block's lanes come in further passes; then the read-outs' norm and gate.
template <typename T, typename TW, typename TO, int KIND, int R>
__global__ __launch_bounds__(1024) void recurrence_tokens_kernel(const RecurrenceIn in, float* __restrict__ state,
                                                                 const float* __restrict__ norm_w, float eps, TO* __restrict__ y,
                                                                 const int* __restrict__ positions, const int* __restrict__ cu,
                                                                 const int* __restrict__ state_slots, int H, int D, int E,
                                                                 int whole_rank) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float scratch[16];
  const int req = blockIdx.y, h = blockIdx.x;
  const int first = cu[req], end = cu[req + 1];
  if (end <= first) return;                  // (the same for the whole block)
  const int tid = threadIdx.x, threads = blockDim.x;
  const int Dl = R * 16;
  float* qs = lds;                           // what meets the state: r, or q times the decay
  float* ks = qs + Dl;
  float* gs = ks + Dl;                       // decays
  float* os = gs + Dl;                       // read-outs, E floats
  float* zs = os + E;                        // kind 1: tanh(z), rank floats
  float* head = state + ((size_t)state_slots[req] * H + h) * E * D;
  const bool whole4 = (D & 3) == 0;
  const float decay = KIND == 0 ? exp2f(in.log2_decay[h]) : 0.f;
  for (int t = first; t < end; ++t) {
    const T* q = (const T*)in.q + (size_t)t * in.ld + (size_t)h * D;
    const T* k = (const T*)in.k + (size_t)t * in.ld + (size_t)h * D;
    float bonus = 0.f;                       // this thread's share of what the token's own k v^T counts for
    // the first columns' state is asked for before anything else
    const bool fresh = t == first && positions[t] == 0;
    const int cols = threads / R, part = tid % R;
    float S[16];
    auto take = [&](int e0) {
      const int e = e0 + tid / R;
      const float* from = head + (size_t)(e < E ? e : 0) * D + part * 4;
      const bool there = !fresh && e < E && tid / R < cols;
#pragma unroll
      for (int i = 0; i < 16; i += 4) {
        const int d = part * 4 + i * R;
        if (whole4) {
          const float4 s4 = (there && d < D) ? *reinterpret_cast<const float4*>(from + i * R) : float4{0.f, 0.f, 0.f, 0.f};
          S[i] = s4.x; S[i + 1] = s4.y; S[i + 2] = s4.z; S[i + 3] = s4.w;
        } else {
#pragma unroll
          for (int j = 0; j < 4; ++j) S[i + j] = (there && d + j < D) ? from[i * R + j] : 0.f;
        }
      }
    };
    take(0);
    // and so are the first columns' value, and the gates and norm weights that the results meet at the end
    const T* v_row = (const T*)in.v + (size_t)t * in.ld + (size_t)h * E;
    const T* g_row = (const T*)in.g + (size_t)t * in.ld + (size_t)h * E;
    const bool column0 = tid / R < cols && tid / R < E;
    const T v_first = v_row[column0 ? tid / R : 0], g_first = g_row[tid < E ? tid : 0];
    const float w_first = norm_w ? norm_w[(size_t)h * E + (tid < E ? tid : 0)] : 1.0f;
    if (KIND == 1) {
      for (int r = tid; r < in.rank; r += threads) zs[r] = tanhf(in.z[(size_t)t * in.z_ld + r]);
      __syncthreads();
      // eight lanes a channel, each four of 32 entries at a time
      for (int x = tid; x < Dl * 8; x += threads) {
        const int d = x >> 3;
        float sum = 0.f, rr = 0.f, kk = 0.f, w0 = 0.f, u = 0.f;
        if (d < D) {
          if ((x & 7) == 0) {
            rr = to_f32(q[d]);
            kk = to_f32(k[d]);
            w0 = in.w0[h * D + d];
            u = in.u[h * D + d];
          }
          const TW* w2 = (const TW*)in.w2 + ((size_t)h * D + d) * in.rank;
#pragma unroll 2
          for (int r = (x & 7) * 4; r < in.rank; r += 32) {
            const floatx4 w = four_of(w2 + r, in.rank - r, whole_rank);
#pragma unroll
            for (int i = 0; i < 4; ++i) sum = fmaf(w[i], r + i < in.rank ? zs[r + i] : 0.f, sum);
          }
        }
        sum += __shfl_xor(sum, 1, NHV_WAVE);
        sum += __shfl_xor(sum, 2, NHV_WAVE);
        sum += __shfl_xor(sum, 4, NHV_WAVE);
        if ((x & 7) == 0) {
          bonus = fmaf(rr * u, kk, bonus);
          qs[d] = rr;
          ks[d] = kk;
          gs[d] = d < D ? exp2_of(-NHV_LOG2E * expf(sum + w0)) : 0.f;
        }
      }
    } else {
      const int half = in.rot / 2;
      for (int d = tid; d < Dl; d += threads) {
        float a = 0.f, b = 0.f;
        if (d < D) {
          a = to_f32(q[d]);
          b = to_f32(k[d]);
          if (d < in.rot) {
            const int i = d < half ? d : d - half;
            float sn, cs;
            nhv_turn_angle<float>(in.turn_positions[t], in.freqs[i], 1.0f, &sn, &cs);
            const float a2 = to_f32(q[d < half ? d + half : i]), b2 = to_f32(k[d < half ? d + half : i]);
            a = d < half ? a * cs - a2 * sn : a * cs + a2 * sn;
            b = d < half ? b * cs - b2 * sn : b * cs + b2 * sn;
          }
          b *= in.k_scale;
          bonus = fmaf(a, b, bonus);
        }
        qs[d] = a * decay;
        ks[d] = b;
        gs[d] = decay;
      }
    }
    bonus = block_sum(bonus, scratch);       // (its barriers also make the vectors visible)
    float ss = 0.f;
    for (int e0 = 0; e0 < E; e0 += cols) {
      const int e = e0 + tid / R;
      const bool column = e < E && tid / R < cols;
      float* mine = head + (size_t)(column ? e : 0) * D + part * 4;
      if (e0 > 0) take(e0);
      const float vv = !column ? 0.f : e0 == 0 ? to_f32(v_first) : to_f32(v_row[e]);
      float sum = 0.f;
#pragma unroll
      for (int i = 0; i < 16; i += 4) {
        const int d = part * 4 + i * R;
        const float4 q4 = *reinterpret_cast<const float4*>(&qs[d]), k4 = *reinterpret_cast<const float4*>(&ks[d]),
                     g4 = *reinterpret_cast<const float4*>(&gs[d]);
        sum = fmaf(q4.x, S[i], fmaf(q4.y, S[i + 1], fmaf(q4.z, S[i + 2], fmaf(q4.w, S[i + 3], sum))));
        S[i] = fmaf(g4.x, S[i], k4.x * vv);
        S[i + 1] = fmaf(g4.y, S[i + 1], k4.y * vv);
        S[i + 2] = fmaf(g4.z, S[i + 2], k4.z * vv);
        S[i + 3] = fmaf(g4.w, S[i + 3], k4.w * vv);
      }
#pragma unroll
      for (int o = 1; o < R; o <<= 1) sum += __shfl_xor(sum, o, NHV_WAVE);
      sum = fmaf(bonus, vv, sum);
      if (column) {
#pragma unroll
        for (int i = 0; i < 16; i += 4) {
          const int d = part * 4 + i * R;
          if (whole4) {
            if (d < D) *reinterpret_cast<float4*>(mine + i * R) = float4{S[i], S[i + 1], S[i + 2], S[i + 3]};
          } else {
#pragma unroll
            for (int j = 0; j < 4; ++j)
              if (d + j < D) mine[i * R + j] = S[i + j];
          }
        }
        if (part == 0) {
          os[e] = sum;
          ss = fmaf(sum, sum, ss);
        }
      }
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)E + eps);
    for (int e = tid; e < E; e += threads) {
      const float z = to_f32(e == tid ? g_first : g_row[e]);
      const float w = e == tid ? w_first : norm_w ? norm_w[(size_t)h * E + e] : 1.0f;
      y[((size_t)t * H + h) * E + e] = from_f32<TO>(os[e] * inv * w * silu_of(z));
    }
    __syncthreads();                         // (the next token's vectors take this one's place)
  }
}

// ---------------------------------------------------------------- the read-out's norm and gate, for many rows
template <typename T, typename TO>
__global__ __launch_bounds__(256) void readout_norm_kernel(const float* __restrict__ o, const T* __restrict__ gate, long long ld,
                                                           const float* __restrict__ w, TO* __restrict__ y, int H, int E,
                                                           float eps, int n_items) {
  const int item = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= n_items) return;
  const int lane = threadIdx.x & 63, t = item / H, h = item % H;
  const float* src = o + (size_t)item * E;
  float ss = 0.f;
  for (int e = lane; e < E; e += NHV_WAVE) ss = fmaf(src[e], src[e], ss);
  const float r = 1.0f / sqrtf(wave_sum(ss) / (float)E + eps);
  for (int e = lane; e < E; e += NHV_WAVE) {
    const float z = to_f32(gate[(size_t)t * ld + (size_t)h * E + e]);
    y[(size_t)item * E + e] = from_f32<TO>(src[e] * r * (w ? w[(size_t)h * E + e] : 1.0f) * silu_of(z));
  }
}

static RecurrenceIn recurrence_in(const void* q, const void* k, const void* v, const void* g, long long ld, const void* log2_decay,
                                  const void* freqs, const void* turn_positions, int rot, float k_scale, const void* z,
                                  long long z_ld, const void* w2, int rank, const void* w0, const void* u) {
  RecurrenceIn in;
  in.q = q; in.k = k; in.v = v; in.g = g; in.ld = ld;
  in.log2_decay = (const float*)log2_decay; in.freqs = (const double*)freqs; in.turn_positions = (const int*)turn_positions;
  in.rot = rot; in.k_scale = k_scale;
  in.z = (const float*)z; in.z_ld = z_ld; in.w2 = w2; in.rank = rank; in.w0 = (const float*)w0; in.u = (const float*)u;
  return in;
}

#define NHV_RECURRENCE_CHECK(name)                                                                                          \
  NHV_REQUIRE(B > 0 && H > 0 && D > 0 && E > 0 && B <= 65535 && H <= 65535, name ": bad sizes B=%d H=%d D=%d E=%d", B, H, D, E); \
  NHV_REQUIRE(D <= 256, name ": key heads of %d entries (up to 256 are taken)", D);                                         \
  NHV_REQUIRE(kind == 0 || kind == 1, name ": kind %d", kind);                                                              \
  NHV_REQUIRE(dtype == NHV_F32 || dtype == NHV_BF16, name ": unknown dtype %d", dtype);                                     \
  NHV_REQUIRE(kind == 1 || (log2_decay && rot >= 0 && rot % 2 == 0 && rot <= D && (rot == 0 || (freqs && turn_positions))),  \
              name ": %d turned entries of %d", rot, D);                                                                    \
  NHV_REQUIRE(kind == 0 || (z && w2 && w0 && u && rank > 0 && z_ld >= rank), name ": decays of rank %d", rank)

// Chunks' places: T / 16 + B + 1. r_out [places, H, 16, Dp], k_out [places, H, Dp, 16], a_out [places, H, 16, 16], decay_out [places, H, Dp], Dp the
// head size rounded up to a multiple of 16.
extern "C" int nhv_recurrence_prepare(int kind, const void* q, const void* k, long long ld, int dtype, const void* log2_decay,
                                      const void* freqs, const void* turn_positions, int rot, float k_scale, const void* z,
                                      long long z_ld, const void* w2, int w2_dtype, int rank, const void* w0, const void* u,
                                      void* r_out, void* k_out, void* a_out, void* decay_out, const void* cu, int B, int H, int D,
                                      int max_q_len, void* stream) {
  const int E = 1;
  NHV_RECURRENCE_CHECK("recurrence_prepare");
  NHV_REQUIRE(max_q_len > 0 && ld >= (long long)H * D, "recurrence_prepare: rows of %lld entries for %d heads of %d", ld, H, D);
  const RecurrenceIn in = recurrence_in(q, k, nullptr, nullptr, ld, log2_decay, freqs, turn_positions, rot, k_scale, z, z_ld, w2,
                                        rank, w0, u);
  const int Dp = (D + 15) / 16 * 16;
  const size_t lds = (size_t)(kind == 1 ? 3 : 2) * NHV_CHUNK * (Dp + 4) * sizeof(float);
  const int chunks = (max_q_len + NHV_CHUNK - 1) / NHV_CHUNK;
  NHV_REQUIRE(chunks <= 65535, "recurrence_prepare: a portion of %d tokens is beyond this kernel's grid", max_q_len);
  const dim3 grid(H, chunks, B);
  const size_t item = dtype == NHV_F32 ? 4 : 2, w_item = w2_dtype == NHV_F32 ? 4 : 2;
  const int whole = D % 4 == 0 && ld % 4 == 0 && (((uintptr_t)q | (uintptr_t)k) % (4 * item)) == 0;
  const int whole_rank = rank % 4 == 0 && (uintptr_t)w2 % (4 * w_item) == 0;
  hipStream_t s = (hipStream_t)stream;
#define LAUNCH(TT, TTW, KIND)                                                                                            \
  hipLaunchKernelGGL((recurrence_prepare_kernel<TT, TTW, KIND>), grid, dim3(256), lds, s, in, (float*)r_out, (float*)k_out, \
                     (float*)a_out, (float*)decay_out, (const int*)cu, H, D, Dp, whole, whole_rank)
  if (kind == 0) { if (dtype == NHV_F32) LAUNCH(float, float, 0); else LAUNCH(bf16_t, bf16_t, 0); }
  else if (w2_dtype == NHV_F32) { if (dtype == NHV_F32) LAUNCH(float, float, 1); else LAUNCH(bf16_t, float, 1); }
  else if (w2_dtype == NHV_BF16) { if (dtype == NHV_F32) LAUNCH(float, bf16_t, 1); else LAUNCH(bf16_t, bf16_t, 1); }
  else return nhv_fail("recurrence_prepare: unknown dtype %d", w2_dtype);
#undef LAUNCH
  NHV_LAUNCH_CHECK("recurrence_prepare");
  return 0;
}

extern "C" int nhv_recurrence_chunks(const void* r_in, const void* k_in, const void* a_in, const void* decay_in, const void* v,
                                     long long ld, int dtype, void* state, void* out, const void* positions, const void* cu,
                                     const void* state_slots, int B, int H, int D, int E, int max_q_len, void* stream) {
  NHV_REQUIRE(B > 0 && H > 0 && D > 0 && E > 0 && B <= 65535 && H <= 65535 && D <= 256 && ld >= (long long)H * E,
              "recurrence_chunks: bad sizes B=%d H=%d D=%d (up to 256) E=%d, rows of %lld", B, H, D, E, ld);
  // (offsets of up to four chunks beyond the portion are counted in 32 bits)
  NHV_REQUIRE(max_q_len > 0 && (max_q_len + 80ll) * ld < (1ll << 31), "recurrence_chunks: a portion of %d rows of %lld entries", max_q_len, ld);
  const int Dp = (D + 15) / 16 * 16, tpw = (Dp / 16 + 3) / 4;
  const dim3 grid(H, (E + 15) / 16, B);
  hipStream_t s = (hipStream_t)stream;
#define LAUNCH(TT, N, EVEN)                                                                                                  \
  hipLaunchKernelGGL((recurrence_chunks_kernel<TT, N, EVEN>), grid, dim3(256), 0, s, (const float*)r_in, (const float*)k_in,    \
                     (const float*)a_in, (const float*)decay_in, (const TT*)v, ld, (float*)state, (float*)out,            \
                     (const int*)positions, (const int*)cu, (const int*)state_slots, H, D, Dp, E)
  const bool even = Dp / 16 == 4 * tpw;
#define BY_EVEN(TT, N) { if (even) LAUNCH(TT, N, true); else LAUNCH(TT, N, false); }
#define BY_TILES(TT)            \
  if (tpw == 1) BY_EVEN(TT, 1)  \
  else if (tpw == 2) BY_EVEN(TT, 2) \
  else if (tpw == 3) BY_EVEN(TT, 3) \
  else BY_EVEN(TT, 4)
  if (dtype == NHV_F32) { BY_TILES(float); }
  else if (dtype == NHV_BF16) { BY_TILES(bf16_t); }
  else return nhv_fail("recurrence_chunks: unknown dtype %d", dtype);
#undef BY_TILES
#undef BY_EVEN
#undef LAUNCH
  NHV_LAUNCH_CHECK("recurrence_chunks");
  return 0;
}

extern "C" int nhv_recurrence_tokens(int kind, const void* q, const void* k, const void* v, const void* g, long long ld, int dtype,
                                     const void* log2_decay, const void* freqs, const void* turn_positions, int rot, float k_scale,
                                     const void* z, long long z_ld, const void* w2, int w2_dtype, int rank, const void* w0,
                                     const void* u, void* state, const void* norm_w, float eps, void* y, int y_dtype,
                                     const void* positions, const void* cu, const void* state_slots, int B, int H, int D, int E,
                                     void* stream) {
  NHV_RECURRENCE_CHECK("recurrence_tokens");
  NHV_REQUIRE(y_dtype == NHV_F32 || y_dtype == NHV_BF16, "recurrence_tokens: unknown dtype %d", y_dtype);
  const RecurrenceIn in = recurrence_in(q, k, v, g, ld, log2_decay, freqs, turn_positions, rot, k_scale, z, z_ld, w2, rank, w0, u);
  int R = 1;
  while (R * 16 < D) R <<= 1;
  int threads = (E * R + 63) / 64 * 64;
  // (with blocks enough for two a compute unit, smaller ones, so that one's loads fall into the other's waits)
  const int most = (long long)B * H >= 512 ? 512 : 1024;
  if (threads > most) threads = most;
  if (threads < 128) threads = 128;
  const size_t lds = (3 * (size_t)R * 16 + E + (kind == 1 ? rank : 0)) * sizeof(float);
  NHV_REQUIRE(lds <= 60 * 1024, "recurrence_tokens: value heads of %d and decays of rank %d are beyond this kernel", E, rank);
  const int whole_rank = rank % 4 == 0 && (uintptr_t)w2 % (w2_dtype == NHV_F32 ? 16 : 8) == 0;
  const dim3 grid(H, B);
  hipStream_t s = (hipStream_t)stream;
#define LAUNCH(TT, TTW, TTO, KIND, RR)                                                                                      \
  hipLaunchKernelGGL((recurrence_tokens_kernel<TT, TTW, TTO, KIND, RR>), grid, dim3(threads), lds, s, in, (float*)state,    \
                     (const float*)norm_w, eps, (TTO*)y, (const int*)positions, (const int*)cu, (const int*)state_slots, H, D, E, whole_rank)
#define BY_R(TT, TTW, TTO, KIND)                       \
  switch (R) {                                         \
    case 1: LAUNCH(TT, TTW, TTO, KIND, 1); break;      \
    case 2: LAUNCH(TT, TTW, TTO, KIND, 2); break;      \
    case 4: LAUNCH(TT, TTW, TTO, KIND, 4); break;      \
    case 8: LAUNCH(TT, TTW, TTO, KIND, 8); break;      \
    default: LAUNCH(TT, TTW, TTO, KIND, 16); break;    \
  }
  const bool f = dtype == NHV_F32, fo = y_dtype == NHV_F32, fw = w2_dtype == NHV_F32;
  if (kind == 0) {
    if (f && fo) { BY_R(float, float, float, 0) }
    else if (!f && !fo) { BY_R(bf16_t, bf16_t, bf16_t, 0) }
    else if (f && !fo) { BY_R(float, bf16_t, bf16_t, 0) }
    else return nhv_fail("recurrence_tokens: bfloat16 rows give bfloat16 rows");
  } else {
    if (f && fo && fw) { BY_R(float, float, float, 1) }
    else if (f && !fo && !fw) { BY_R(float, bf16_t, bf16_t, 1) }
    else if (!f && !fo && !fw) { BY_R(bf16_t, bf16_t, bf16_t, 1) }
    else return nhv_fail("recurrence_tokens: rows, weights and results of types %d, %d, %d are not taken", dtype, w2_dtype, y_dtype);
  }
#undef BY_R
#undef LAUNCH
  NHV_LAUNCH_CHECK("recurrence_tokens");
  return 0;
}

extern "C" int nhv_readout_norm(const void* o, const void* gate, long long ld, int gate_dtype, const void* w, void* y, int y_dtype,
                                int T, int H, int E, float eps, void* stream) {
  NHV_REQUIRE(T > 0 && H > 0 && E > 0 && (long long)T * H < (1ll << 31) && ld >= (long long)H * E,
              "readout_norm: bad sizes T=%d H=%d E=%d, gate rows of %lld", T, H, E, ld);
  const int n_items = T * H;
  const dim3 grid((unsigned)((n_items + 3) / 4));
  hipStream_t s = (hipStream_t)stream;
#define LAUNCH(TT, TTO)                                                                                                    \
  hipLaunchKernelGGL((readout_norm_kernel<TT, TTO>), grid, dim3(256), 0, s, (const float*)o, (const TT*)gate, ld,          \
                     (const float*)w, (TTO*)y, H, E, eps, n_items)
  if (gate_dtype == NHV_F32 && y_dtype == NHV_F32) LAUNCH(float, float);
  else if (gate_dtype == NHV_F32 && y_dtype == NHV_BF16) LAUNCH(float, bf16_t);
  else if (gate_dtype == NHV_BF16 && y_dtype == NHV_BF16) LAUNCH(bf16_t, bf16_t);
  else return nhv_fail("readout_norm: gates of type %d and rows of type %d are not taken together", gate_dtype, y_dtype);
#undef LAUNCH
  NHV_LAUNCH_CHECK("readout_norm");
  return 0;
}
