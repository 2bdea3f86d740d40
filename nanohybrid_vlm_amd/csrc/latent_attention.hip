// Kernels of attention over a cached latent: every token stores one row [c | r], c the normed low-rank latent that
// keys and values of all heads are made of, r a rotated key part shared by all heads (it may be absent).
//   nhv_latent_prepare      the packed down projections of a step's rows -> the normed query latent (if there is one), and
//                           the row [RMS-normed c | rotated r] stored at the step's slots
//   nhv_head_gemm           y[t, h, :] = M_h x[t, h, :] for a matrix per head (strides say which way M_h lies), with an
//                           optional sigmoid gate on the result, one per (token, head) or one per entry
//   nhv_head_gemm_fewrows   the same for up to 16 rows, with the turning of the queries' rotated part in the same launch
//   nhv_head_gemm_bf16      the same on the matrix cores for any number of rows, turning included
//   nhv_rotate_heads        the rotated part of every query head, turned by position and copied beside the rest
// Pairs (2i, 2i + 1), or (i, i + r / 2) of the r rotated entries where ``halves`` is set, turn by angle = position *
// freqs[i]; cosine and sine are multiplied by ``gain``. The frequencies
// come as doubles and the product with the position is taken and brought into [-pi, pi] in double (a float product
// of a position in the thousands is off by 1e-4 of a turn), then sine and cosine are taken. Norm statistics and sums
// are float; rows are float or bfloat16.
#include "nhv_common.h"
#include "nhv_rotation.h"
#include <math.h>

// entries of the rotated part that pair p is made of
__device__ __forceinline__ int nhv_pair_first(int p, int rot, int halves) { return halves ? p : 2 * p; }
__device__ __forceinline__ int nhv_pair_second(int p, int rot, int halves) { return halves ? p + rot / 2 : 2 * p + 1; }

// The gate on entry n of head h's result at row m: none (null), mode 1: one float per (row, head), gate[m gs_t + h];
// mode 2: one per entry, of the rows' type, gate[m gs_t + h N + n].
template <typename T>
__device__ __forceinline__ float nhv_head_gate_of(const void* gate, int mode, long long gs_t, int m, int h, int N, int n) {
  const float z = mode == 2 ? to_f32(reinterpret_cast<const T*>(gate)[(size_t)m * gs_t + (size_t)h * N + n])
                            : reinterpret_cast<const float*>(gate)[(size_t)m * gs_t + h];
  return 1.0f / (1.0f + expf(-z));
}

// Pair p of head h at row t, turned from x (entry x_rot_off on) into y (entry y_rot_off on).
template <typename T>
__device__ __forceinline__ void nhv_turn_pair(const T* s, T* d, int p, int rot, int halves, int pos, const double* freqs, float gain) {
  float sn, cs;
  nhv_turn_angle<T>(pos, freqs[p], gain, &sn, &cs);
  const int a = nhv_pair_first(p, rot, halves), b = nhv_pair_second(p, rot, halves);
  const float u = to_f32(s[a]), v = to_f32(s[b]);
  d[a] = from_f32<T>(u * cs - v * sn);
  d[b] = from_f32<T>(v * cs + u * sn);
}

// a: [T, A] rows of type TA. Query latent (q_rank > 0): columns q_off .. q_off + q_rank, normed with wq into cq [T, q_rank]. Latent:
// columns c_off .. c_off + kv_rank normed with wc, then ``rot`` columns turned; both stored at slot_mapping[t] in
// ``cache`` (rows of ``row`` entries; entries beyond kv_rank + rot become zeros). kv_rank 0: nothing is stored.
template <typename T, typename TA>
__global__ void latent_prepare_kernel(const TA* __restrict__ a, int A, int q_off, int q_rank, int c_off, int kv_rank,
                                      int rot, const float* __restrict__ wq, const float* __restrict__ wc, float eps,
                                      const double* __restrict__ freqs, float gain, const int* __restrict__ positions,
                                      const int* __restrict__ slot_mapping, T* __restrict__ cache, int row,
                                      T* __restrict__ cq, int halves) {
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  const TA* src = a + (size_t)t * A;
  float ss = 0.f;
  if (q_rank > 0) {                          // the same for the whole grid
    for (int i = threadIdx.x; i < q_rank; i += blockDim.x) {
      const float v = to_f32(src[q_off + i]);
      ss += v * v;
    }
    const float rq = 1.0f / sqrtf(block_sum(ss, scratch) / (float)q_rank + eps);
    for (int i = threadIdx.x; i < q_rank; i += blockDim.x)
      cq[(size_t)t * q_rank + i] = from_f32<T>(to_f32(src[q_off + i]) * rq * wq[i]);
  }
  if (kv_rank == 0 || slot_mapping == nullptr) return;
  const int slot = slot_mapping[t];          // the same for the whole block
  if (slot < 0) return;
  ss = 0.f;
  for (int i = threadIdx.x; i < kv_rank; i += blockDim.x) {
    const float v = to_f32(src[c_off + i]);
    ss += v * v;
  }
  const float rc = 1.0f / sqrtf(block_sum(ss, scratch) / (float)kv_rank + eps);
  T* dst = cache + (size_t)slot * row;
  for (int i = threadIdx.x; i < kv_rank; i += blockDim.x) dst[i] = from_f32<T>(to_f32(src[c_off + i]) * rc * wc[i]);
  const int pos = positions[t];
  for (int i = threadIdx.x; i < rot / 2; i += blockDim.x) {
    float sn, cs;
    nhv_turn_angle<T>(pos, freqs[i], gain, &sn, &cs);
    const int first = nhv_pair_first(i, rot, halves), second = nhv_pair_second(i, rot, halves);
    const float u = to_f32(src[c_off + kv_rank + first]), v = to_f32(src[c_off + kv_rank + second]);
    dst[kv_rank + first] = from_f32<T>(u * cs - v * sn);
    dst[kv_rank + second] = from_f32<T>(v * cs + u * sn);
  }
  // (entries of the row beyond the rotated part: zeros, which meet zeros in the queries)
  for (int i = kv_rank + rot + threadIdx.x; i < row; i += blockDim.x) dst[i] = from_f32<T>(0.f);
}

extern "C" int nhv_latent_prepare(const void* a, int a_dtype, int A, int q_off, int q_rank, int c_off, int kv_rank, int rot,
                                  const void* wq, const void* wc, float eps, const void* freqs, float gain,
                                  const void* positions, const void* slot_mapping, void* cache, int row, void* cq, int halves,
                                  int T, int dtype, void* stream) {
  NHV_REQUIRE(T > 0 && A > 0 && q_rank >= 0 && kv_rank >= 0 && q_rank + kv_rank > 0 && rot >= 0 && rot % 2 == 0,
              "latent_prepare: bad sizes T=%d A=%d q_rank=%d kv_rank=%d rot=%d", T, A, q_rank, kv_rank, rot);
  NHV_REQUIRE((q_rank == 0 || (q_off >= 0 && q_off + q_rank <= A)) && (kv_rank == 0 || (c_off >= 0 && c_off + kv_rank + rot <= A)),
              "latent_prepare: columns %d+%d and %d+%d+%d of %d", q_off, q_rank, c_off, kv_rank, rot, A);
  NHV_REQUIRE(kv_rank == 0 || slot_mapping == nullptr || (cache != nullptr && row >= kv_rank + rot),
              "latent_prepare: cache rows of %d entries for %d + %d", row, kv_rank, rot);
  NHV_REQUIRE(rot == 0 || kv_rank == 0 || freqs != nullptr, "latent_prepare: a rotated part without frequencies");
  hipStream_t s = (hipStream_t)stream;
#define LAUNCH(TT, TA)                                                                                                     \
  hipLaunchKernelGGL((latent_prepare_kernel<TT, TA>), dim3(T), dim3(256), 0, s, (const TA*)a, A, q_off, q_rank, c_off,      \
                     kv_rank, rot, (const float*)wq, (const float*)wc, eps, (const double*)freqs, gain,                    \
                     (const int*)positions, (const int*)slot_mapping, (TT*)cache, row, (TT*)cq, halves)
  if (dtype == NHV_F32 && a_dtype == NHV_F32) LAUNCH(float, float);
  else if (dtype == NHV_BF16 && a_dtype == NHV_F32) LAUNCH(bf16_t, float);
  else if (dtype == NHV_BF16 && a_dtype == NHV_BF16) LAUNCH(bf16_t, bf16_t);
  else return nhv_fail("latent_prepare: unknown dtypes %d, %d", a_dtype, dtype);
#undef LAUNCH
  NHV_LAUNCH_CHECK("latent_prepare");
  return 0;
}

// ---------------------------------------------------------------- a matrix per head
// y[t * ys_t + h * ys_h + n] = sum over k of x[t * xs_t + h * xs_h + k] * w[h * ws_h + n * ws_n + k * ws_k], k rising,
// one thread per output, so a row's result does not depend on its batch. A block owns 32 rows x 64 outputs of one head
// and walks over k in pieces of 16 through LDS. gate: y *= the sigmoid of a gate (nhv_head_gate_of).
#define HG_TM 32
#define HG_TN 64
#define HG_TK 16
template <typename T>
__global__ __launch_bounds__(256) void head_gemm_kernel(const T* __restrict__ x, long long xs_t, long long xs_h,
                                                        const T* __restrict__ w, long long ws_h, long long ws_n,
                                                        long long ws_k, T* __restrict__ y, long long ys_t, long long ys_h,
                                                        const void* __restrict__ gate, int gate_mode, long long gs_t,
                                                        int rows, int N, int K) {
  __shared__ float xs[HG_TM][HG_TK];
  __shared__ float wt[HG_TN][HG_TK + 1];
  const int h = blockIdx.z;
  const int m0 = blockIdx.x * HG_TM, n0 = blockIdx.y * HG_TN;
  const int tx = threadIdx.x & 63, ty = threadIdx.x >> 6;
  float acc[HG_TM / 4];
#pragma unroll
  for (int i = 0; i < HG_TM / 4; ++i) acc[i] = 0.f;
  const T* xh = x + (size_t)h * xs_h;
  const T* wh = w + (size_t)h * ws_h;
  for (int k0 = 0; k0 < K; k0 += HG_TK) {
    for (int idx = threadIdx.x; idx < HG_TM * HG_TK; idx += 256) {
      const int m = idx / HG_TK, kk = idx % HG_TK;
      xs[m][kk] = (m0 + m < rows && k0 + kk < K) ? to_f32(xh[(size_t)(m0 + m) * xs_t + k0 + kk]) : 0.f;
    }
    for (int idx = threadIdx.x; idx < HG_TN * HG_TK; idx += 256) {
      int n, kk;
      if (ws_k == 1) { n = idx / HG_TK; kk = idx % HG_TK; }
      else { n = idx % HG_TN; kk = idx / HG_TN; }
      wt[n][kk] = (n0 + n < N && k0 + kk < K) ? to_f32(wh[(size_t)(n0 + n) * ws_n + (size_t)(k0 + kk) * ws_k]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < HG_TK; ++kk) {
      const float wv = wt[tx][kk];
#pragma unroll
      for (int i = 0; i < HG_TM / 4; ++i) acc[i] = fmaf(xs[ty * (HG_TM / 4) + i][kk], wv, acc[i]);
    }
    __syncthreads();
  }
  const int n = n0 + tx;
  if (n >= N) return;
#pragma unroll
  for (int i = 0; i < HG_TM / 4; ++i) {
    const int m = m0 + ty * (HG_TM / 4) + i;
    if (m >= rows) continue;
    float v = acc[i];
    if (gate != nullptr) v *= nhv_head_gate_of<T>(gate, gate_mode, gs_t, m, h, N, n);
    y[(size_t)m * ys_t + (size_t)h * ys_h + n] = from_f32<T>(v);
  }
}

extern "C" int nhv_head_gemm(const void* x, long long xs_t, long long xs_h, const void* w, long long ws_h, long long ws_n,
                             long long ws_k, void* y, long long ys_t, long long ys_h, const void* gate, int gate_mode,
                             long long gs_t, int rows, int H, int N, int K, int dtype, void* stream) {
  NHV_REQUIRE(rows > 0 && H > 0 && N > 0 && K > 0 && H <= 65535, "head_gemm: bad sizes rows=%d H=%d N=%d K=%d", rows, H, N, K);
  const dim3 grid((rows + HG_TM - 1) / HG_TM, (N + HG_TN - 1) / HG_TN, H);
  NHV_REQUIRE(grid.y <= 65535, "head_gemm: %d outputs a head are too many", N);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == NHV_F32)
    hipLaunchKernelGGL(head_gemm_kernel<float>, grid, dim3(256), 0, s, (const float*)x, xs_t, xs_h, (const float*)w, ws_h,
                       ws_n, ws_k, (float*)y, ys_t, ys_h, gate, gate_mode, gs_t, rows, N, K);
  else if (dtype == NHV_BF16)
    hipLaunchKernelGGL(head_gemm_kernel<bf16_t>, grid, dim3(256), 0, s, (const bf16_t*)x, xs_t, xs_h, (const bf16_t*)w,
                       ws_h, ws_n, ws_k, (bf16_t*)y, ys_t, ys_h, gate, gate_mode, gs_t, rows, N, K);
  else
    return nhv_fail("head_gemm: unknown dtype %d", dtype);
  NHV_LAUNCH_CHECK("head_gemm");
  return 0;
}

// The same for up to 16 rows (a decoding step): a block owns 64 outputs of one head. It first brings the head's rows
// of x (as floats) and its 64 x K piece of the matrix into LDS, every thread asking for all its share at once (a
// thread that walked over k with loads from memory waited for memory at every step); then lane = output, wave = four
// of the rows, k rising as above, so the sums are the same bits. One more block a head may turn the rotated part of x
// and copy it beside the outputs (``rot`` entries from x_rot_off to y_rot_off), which saves the launch of
// nhv_rotate_heads.
template <typename V>
__device__ __forceinline__ void hg_load8f(const V* p, float* out);
template <>
__device__ __forceinline__ void hg_load8f<bf16_t>(const bf16_t* p, float* out) {
  typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 v8;
  const v8 v = *reinterpret_cast<const v8*>(p);
#pragma unroll
  for (int e = 0; e < 8; ++e) out[e] = (float)v[e];
}
template <>
__device__ __forceinline__ void hg_load8f<float>(const float* p, float* out) {
  const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
  out[0] = a.x; out[1] = a.y; out[2] = a.z; out[3] = a.w; out[4] = b.x; out[5] = b.y; out[6] = b.z; out[7] = b.w;
}

// VEC: K and N are multiples of 8 and every row of x and of the matrix starts at a multiple of 8 entries from an
// address that is a multiple of 32 bytes (the host checks), so eight entries can be asked for at once.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void head_gemm_fewrows_kernel(const T* __restrict__ x, long long xs_t, long long xs_h,
                                                                const T* __restrict__ w, long long ws_h, long long ws_n,
                                                                long long ws_k, T* __restrict__ y, long long ys_t,
                                                                long long ys_h, const void* __restrict__ gate, int gate_mode,
                                                                long long gs_t, int rows, int N, int K, int n_chunks, int rot,
                                                                int x_rot_off, int y_rot_off, int halves,
                                                                const double* __restrict__ freqs,
                                                                float gain, const int* __restrict__ positions) {
  extern __shared__ float xs[];              // 16 x K floats, then the block's piece of the matrix
  const int h = blockIdx.y;
  if ((int)blockIdx.x == n_chunks) {         // the rotated part
    for (int i = threadIdx.x; i < rows * (rot / 2); i += blockDim.x) {
      const int t = i / (rot / 2), p = i % (rot / 2);
      nhv_turn_pair(x + (size_t)t * xs_t + (size_t)h * xs_h + x_rot_off, y + (size_t)t * ys_t + (size_t)h * ys_h + y_rot_off, p,
                    rot, halves, positions[t], freqs, gain);
    }
    return;
  }
  // [K][LDW]: rows a little longer than 64 outputs: pieces of 16 bytes stay aligned, and threads that walk along k (a
  // matrix that is contiguous in k) do not all store into one bank
  constexpr int LDW = 64 + 16 / (int)sizeof(T);
  T* wl = reinterpret_cast<T*>(xs + 16 * K);
  const int n0 = blockIdx.x * 64;
  const T* wh = w + (size_t)h * ws_h;
  const T* xh = x + (size_t)h * xs_h;
  if (VEC) {
    // eight entries a load, and all of a thread's loads asked for before the first is stored (the matrix comes from
    // memory: a thread that stored each piece before it asked for the next waited once a piece)
    const int w_chunks = 8 * K;              // 64 x K / 8
    for (int c0 = 0; c0 < w_chunks; c0 += 256 * 8) {
      float v[8][8];
#pragma unroll
      for (int b = 0; b < 8; ++b) {
        const int c = c0 + b * 256 + (int)threadIdx.x;
        if (c >= w_chunks) continue;
        int n, k;
        if (ws_k == 1) { n = c / (K / 8); k = (c % (K / 8)) * 8; }
        else { k = c / 8; n = (c % 8) * 8; }
        const bool ok = ws_k == 1 ? n0 + n < N : n0 + n + 7 < N;
        if (ok) hg_load8f(wh + (size_t)(n0 + n) * ws_n + (size_t)k * ws_k, v[b]);
        else {
#pragma unroll
          for (int i = 0; i < 8; ++i) v[b][i] = (ws_k != 1 && n0 + n + i < N) ? to_f32(wh[(size_t)(n0 + n + i) + (size_t)k * ws_k]) : 0.f;
        }
      }
#pragma unroll
      for (int b = 0; b < 8; ++b) {
        const int c = c0 + b * 256 + (int)threadIdx.x;
        if (c >= w_chunks) continue;
        if (ws_k == 1) {
          const int n = c / (K / 8), k = (c % (K / 8)) * 8;
#pragma unroll
          for (int i = 0; i < 8; ++i) wl[(k + i) * LDW + n] = from_f32<T>(v[b][i]);
        } else {
          const int k = c / 8, n = (c % 8) * 8;
#pragma unroll
          for (int i = 0; i < 8; ++i) wl[k * LDW + n + i] = from_f32<T>(v[b][i]);
        }
      }
    }
    const int x_chunks = 2 * K;              // 16 x K / 8
    for (int c = threadIdx.x; c < x_chunks; c += blockDim.x) {
      const int t = c / (K / 8), k = (c % (K / 8)) * 8;
      float v[8];
      if (t < rows) hg_load8f(xh + (size_t)t * xs_t + k, v);
#pragma unroll
      for (int i = 0; i < 8; ++i) xs[t * K + k + i] = t < rows ? v[i] : 0.f;
    }
  } else {
    if (ws_k == 1) {                         // a row of the matrix is contiguous in k: threads walk along k
      for (int i = threadIdx.x; i < 64 * K; i += blockDim.x) {
        const int n = i / K, k = i % K;
        wl[k * LDW + n] = n0 + n < N ? wh[(size_t)(n0 + n) * ws_n + k] : from_f32<T>(0.f);
      }
    } else {                                 // contiguous in n
      for (int i = threadIdx.x; i < 64 * K; i += blockDim.x) {
        const int k = i / 64, n = i % 64;
        wl[k * LDW + n] = n0 + n < N ? wh[(size_t)(n0 + n) * ws_n + (size_t)k * ws_k] : from_f32<T>(0.f);
      }
    }
    for (int i = threadIdx.x; i < 16 * K; i += blockDim.x) {
      const int t = i / K, k = i % K;
      xs[i] = t < rows ? to_f32(xh[(size_t)t * xs_t + k]) : 0.f;
    }
  }
  __syncthreads();
  const int lane = threadIdx.x & 63, t0 = (threadIdx.x >> 6) * 4;
  const int n = n0 + lane;
  if (n >= N || t0 >= rows) return;
  float acc[4] = {0.f, 0.f, 0.f, 0.f};
  const float* x0 = xs + t0 * K;
  for (int k = 0; k < K; ++k) {
    const float wv = to_f32(wl[k * LDW + lane]);
#pragma unroll
    for (int t = 0; t < 4; ++t) acc[t] = fmaf(x0[t * K + k], wv, acc[t]);
  }
#pragma unroll
  for (int t = 0; t < 4; ++t) {
    if (t0 + t >= rows) break;
    float v = acc[t];
    if (gate != nullptr) v *= nhv_head_gate_of<T>(gate, gate_mode, gs_t, t0 + t, h, N, n);
    y[(size_t)(t0 + t) * ys_t + (size_t)h * ys_h + n] = from_f32<T>(v);
  }
}

extern "C" int nhv_head_gemm_fewrows(const void* x, long long xs_t, long long xs_h, const void* w, long long ws_h,
                                     long long ws_n, long long ws_k, void* y, long long ys_t, long long ys_h, const void* gate,
                                     int gate_mode, long long gs_t, int rows, int H, int N, int K, int rot, int x_rot_off,
                                     int y_rot_off, int halves, const void* freqs, float gain, const void* positions, int dtype, void* stream) {
  const size_t item = dtype == NHV_F32 ? 4 : 2;
  const size_t lds = 16 * (size_t)K * sizeof(float) + (64 + 16 / item) * (size_t)K * item;
  NHV_REQUIRE(rows > 0 && rows <= 16 && H > 0 && H <= 65535 && N > 0 && K > 0 && lds <= 96 * 1024,
              "head_gemm_fewrows: bad sizes rows=%d (up to 16) H=%d N=%d K=%d (LDS of %zu bytes, up to 98304)", rows, H, N, K, lds);
  NHV_REQUIRE(rot >= 0 && rot % 2 == 0 && (rot == 0 || (freqs != nullptr && positions != nullptr)),
              "head_gemm_fewrows: a rotated part of %d entries needs frequencies and positions", rot);
  const int n_chunks = (N + 63) / 64;
  const dim3 grid(n_chunks + (rot > 0 ? 1 : 0), H);
  hipStream_t s = (hipStream_t)stream;
  const long long strides[] = {xs_t, xs_h, ws_h, ws_n == 1 ? ws_k : ws_n};
  bool vec = K % 8 == 0 && N % 8 == 0 && (uintptr_t)x % 32 == 0 && (uintptr_t)w % 32 == 0 && (ws_n == 1 || ws_k == 1);
  for (long long st : strides) vec = vec && st % 8 == 0;
#define NHV_HG_LAUNCH(TYPE, VEC)                                                                                          \
  do {                                                                                                                    \
    if (lds > 64 * 1024)                                                                                                  \
      (void)hipFuncSetAttribute((const void*)head_gemm_fewrows_kernel<TYPE, VEC>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); \
    hipLaunchKernelGGL((head_gemm_fewrows_kernel<TYPE, VEC>), grid, dim3(256), lds, s, (const TYPE*)x, xs_t, xs_h,          \
                       (const TYPE*)w, ws_h, ws_n, ws_k, (TYPE*)y, ys_t, ys_h, gate, gate_mode, gs_t, rows, N, K, n_chunks,   \
                       rot, x_rot_off, y_rot_off, halves, (const double*)freqs, gain, (const int*)positions);                      \
  } while (0)
  if (dtype == NHV_F32) {
    if (vec) NHV_HG_LAUNCH(float, true); else NHV_HG_LAUNCH(float, false);
  } else if (dtype == NHV_BF16) {
    if (vec) NHV_HG_LAUNCH(bf16_t, true); else NHV_HG_LAUNCH(bf16_t, false);
  } else {
    return nhv_fail("head_gemm_fewrows: unknown dtype %d", dtype);
  }
#undef NHV_HG_LAUNCH
  NHV_LAUNCH_CHECK("head_gemm_fewrows");
  return 0;
}

// ---------------------------------------------------------------- a matrix per head on the matrix cores
// The same in bfloat16 for matrices that are contiguous in k (M_h[n, k] = w[h N K + n K + k]), any number of rows, K and
// every stride a multiple of 8 and every start 16 bytes aligned (the host checks). A wave owns MT x 16 rows and NT x 16
// outputs of one head; the matrix rows are the 16 x 32 operand and the rows of x the 32 x 16 one, both asked for from
// memory in the operands' own layout, 16 bytes a lane (a head's matrix is small and is found in L2 by all but the first
// rows' blocks). A lane then holds four consecutive outputs of one row. Sums run over k in rising order whatever MT and
// NT are, so a row's result does not depend on how many rows there are. One more block of outputs turns the rotated part.
typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 hg_bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(__bf16)))) __bf16 hg_bf16x4;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float hg_floatx4;

// U: steps of 32 columns whose loads are all under way before the first product.
template <int MT, int NT, int WAVES, int U>
__global__ __launch_bounds__(64 * WAVES) void head_gemm_mfma_kernel(const bf16_t* __restrict__ x, long long xs_t, long long xs_h,
                                                                    const bf16_t* __restrict__ w, bf16_t* __restrict__ y,
                                                                    long long ys_t, long long ys_h,
                                                                    const void* __restrict__ gate, int gate_mode,
                                                                    long long gs_t, int rows, int N, int K, int n_chunks, int rot,
                                                                    int x_rot_off, int y_rot_off, int halves,
                                                                    const double* __restrict__ freqs, float gain,
                                                                    const int* __restrict__ positions) {
  const int h = blockIdx.z;
  const int m0 = blockIdx.y * 16 * MT;
  if ((int)blockIdx.x == n_chunks) {         // the rotated part of these rows
    const int here = min(16 * MT, rows - m0), half = rot / 2;
    for (int i = threadIdx.x; i < here * half; i += 64 * WAVES) {
      const int t = m0 + i / half;
      nhv_turn_pair(x + (size_t)t * xs_t + (size_t)h * xs_h + x_rot_off, y + (size_t)t * ys_t + (size_t)h * ys_h + y_rot_off,
                    i % half, rot, halves, positions[t], freqs, gain);
    }
    return;
  }
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int col = lane & 15, grp = lane >> 4;
  const int n0 = (blockIdx.x * WAVES + wave) * 16 * NT;
  if (n0 >= N) return;
  const bf16_t* wrow[NT];
  bool n_ok[NT];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) {
    const int n = n0 + nt * 16 + col;
    n_ok[nt] = n < N;
    wrow[nt] = w + ((size_t)h * N + (n_ok[nt] ? n : 0)) * K;
  }
  const bf16_t* xrow[MT];
  bool m_ok[MT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    const int m = m0 + mt * 16 + col;
    m_ok[mt] = m < rows;
    xrow[mt] = x + (size_t)(m_ok[mt] ? m : 0) * xs_t + (size_t)h * xs_h;
  }
  hg_floatx4 acc[MT][NT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt)
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) acc[mt][nt] = hg_floatx4{0.f, 0.f, 0.f, 0.f};
  hg_bf16x8 zero;
#pragma unroll
  for (int i = 0; i < 8; ++i) zero[i] = (__bf16)0.f;
  for (int k0 = 0; k0 < K; k0 += 32 * U) {
    hg_bf16x8 a[U][NT], b[U][MT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + u * 32 + grp * 8;
      const bool k_ok = k < K;               // K is a multiple of 8: a piece is inside or outside as a whole
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) a[u][nt] = (n_ok[nt] && k_ok) ? *reinterpret_cast<const hg_bf16x8*>(wrow[nt] + k) : zero;
#pragma unroll
      for (int mt = 0; mt < MT; ++mt) b[u][mt] = (m_ok[mt] && k_ok) ? *reinterpret_cast<const hg_bf16x8*>(xrow[mt] + k) : zero;
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int mt = 0; mt < MT; ++mt)
#pragma unroll
        for (int nt = 0; nt < NT; ++nt)
          acc[mt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[u][nt], b[u][mt], acc[mt][nt], 0, 0, 0);
  }
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    const int m = m0 + mt * 16 + col;
    if (!m_ok[mt]) continue;
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      const int n = n0 + nt * 16 + grp * 4;
      float v[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        v[j] = acc[mt][nt][j];
        if (gate != nullptr && n + j < N) v[j] *= nhv_head_gate_of<bf16_t>(gate, gate_mode, gs_t, m, h, N, n + j);
      }
      bf16_t* dst = y + (size_t)m * ys_t + (size_t)h * ys_h + n;
      if (n + 3 < N && ((uintptr_t)dst & 7) == 0) {
        hg_bf16x4 four;
#pragma unroll
        for (int j = 0; j < 4; ++j) four[j] = (__bf16)v[j];
        *reinterpret_cast<hg_bf16x4*>(dst) = four;
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (n + j < N) dst[j] = (bf16_t)v[j];
      }
    }
  }
}

// The same for many rows (K <= HT_MAX_K): a block owns 64 rows of one head and walks over all of its outputs, 128 at a time.
// The rows come into LDS once, whole rows of K entries; a wave takes 32 of the 128 outputs, with the matrix rows straight
// from memory (L2), and the results go back through LDS so that rows are written in pieces of 16 bytes side by side.
#define HT_ROWS 64
#define HT_COLS 128
#define HT_MAX_K 512
template <int U>
__global__ __launch_bounds__(256) void head_gemm_tile_kernel(const bf16_t* __restrict__ x, long long xs_t, long long xs_h,
                                                             const bf16_t* __restrict__ w, bf16_t* __restrict__ y,
                                                             long long ys_t, long long ys_h, const void* __restrict__ gate,
                                                             int gate_mode, long long gs_t, int rows, int N, int K, int rot,
                                                             int x_rot_off, int y_rot_off, int halves,
                                                             const double* __restrict__ freqs, float gain,
                                                             const int* __restrict__ positions, int vec_out, int vec_gate) {
  extern __shared__ __attribute__((aligned(16))) unsigned char ht_lds[];
  const int pitch = K + 8;                               // 16 bytes more than a row: the rows spread over the banks
  bf16_t* xs = reinterpret_cast<bf16_t*>(ht_lds);        // [64][pitch]
  constexpr int YP = HT_COLS + 8;
  bf16_t* ys = xs + HT_ROWS * pitch;                     // [64][YP]
  const int h = blockIdx.x, m0 = blockIdx.y * HT_ROWS;
  const int here = min(HT_ROWS, rows - m0);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int col = lane & 15, grp = lane >> 4;
  const int pieces = K / 8;
  for (int i = threadIdx.x; i < HT_ROWS * pieces; i += 256) {
    const int m = i / pieces, p = i % pieces;
    hg_bf16x8 v;
    if (m < here) v = *reinterpret_cast<const hg_bf16x8*>(x + (size_t)(m0 + m) * xs_t + (size_t)h * xs_h + p * 8);
    else {
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = (__bf16)0.f;
    }
    *reinterpret_cast<hg_bf16x8*>(xs + m * pitch + p * 8) = v;
  }
  // the rotated part of these rows, while the rows are on their way
  for (int i = threadIdx.x; i < here * (rot / 2); i += 256) {
    const int t = m0 + i / (rot / 2);
    nhv_turn_pair(x + (size_t)t * xs_t + (size_t)h * xs_h + x_rot_off, y + (size_t)t * ys_t + (size_t)h * ys_h + y_rot_off,
                  i % (rot / 2), rot, halves, positions[t], freqs, gain);
  }
  hg_bf16x8 zero;
#pragma unroll
  for (int i = 0; i < 8; ++i) zero[i] = (__bf16)0.f;
  __syncthreads();
  for (int c0 = 0; c0 < N; c0 += HT_COLS) {
    const int n0 = c0 + wave * 32;
    if (n0 < N) {                                        // the whole wave; every wave meets the barriers below
      const bf16_t* wrow[2];
      bool n_ok[2];
#pragma unroll
      for (int nt = 0; nt < 2; ++nt) {
        const int n = n0 + nt * 16 + col;
        n_ok[nt] = n < N;
        wrow[nt] = w + ((size_t)h * N + (n_ok[nt] ? n : 0)) * K;
      }
      hg_floatx4 acc[4][2];
#pragma unroll
      for (int mt = 0; mt < 4; ++mt)
#pragma unroll
        for (int nt = 0; nt < 2; ++nt) acc[mt][nt] = hg_floatx4{0.f, 0.f, 0.f, 0.f};
      // gates of four entries at once, asked for before the products
      hg_bf16x4 g4[4][2];
      if (vec_gate) {
#pragma unroll
        for (int mt = 0; mt < 4; ++mt)
#pragma unroll
          for (int nt = 0; nt < 2; ++nt) {
            const int n = n0 + nt * 16 + grp * 4, m = m0 + min(mt * 16 + col, here - 1);
            g4[mt][nt] = *reinterpret_cast<const hg_bf16x4*>(reinterpret_cast<const bf16_t*>(gate) + (size_t)m * gs_t + (size_t)h * N +
                                                             (n < N ? n : 0));
          }
      }
      for (int k0 = 0; k0 < K; k0 += 32 * U) {
        hg_bf16x8 a[U][2];
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int k = k0 + u * 32 + grp * 8;
#pragma unroll
          for (int nt = 0; nt < 2; ++nt) a[u][nt] = (n_ok[nt] && k < K) ? *reinterpret_cast<const hg_bf16x8*>(wrow[nt] + k) : zero;
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int k = k0 + u * 32 + grp * 8;
#pragma unroll
          for (int mt = 0; mt < 4; ++mt) {
            const hg_bf16x8 b = k < K ? *reinterpret_cast<const hg_bf16x8*>(xs + (mt * 16 + col) * pitch + k) : zero;
#pragma unroll
            for (int nt = 0; nt < 2; ++nt) acc[mt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[u][nt], b, acc[mt][nt], 0, 0, 0);
          }
        }
      }
#pragma unroll
      for (int mt = 0; mt < 4; ++mt)
#pragma unroll
        for (int nt = 0; nt < 2; ++nt) {
          hg_bf16x4 four;
          float v[4];
#pragma unroll
          for (int j = 0; j < 4; ++j) v[j] = acc[mt][nt][j];
          if (vec_gate) {
#pragma unroll
            for (int j = 0; j < 4; ++j)
              v[j] *= __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * (float)g4[mt][nt][j]));
          } else if (gate != nullptr && mt * 16 + col < here) {
            const int n = n0 + nt * 16 + grp * 4;
#pragma unroll
            for (int j = 0; j < 4; ++j)
              if (n + j < N) v[j] *= nhv_head_gate_of<bf16_t>(gate, gate_mode, gs_t, m0 + mt * 16 + col, h, N, n + j);
          }
#pragma unroll
          for (int j = 0; j < 4; ++j) four[j] = (__bf16)v[j];
          *reinterpret_cast<hg_bf16x4*>(ys + (mt * 16 + col) * YP + wave * 32 + nt * 16 + grp * 4) = four;
        }
    }
    __syncthreads();
    const int width = min(HT_COLS, N - c0);
    if (vec_out) {                                       // N and the rows of y are pieces of 16 bytes
      for (int i = threadIdx.x; i < here * (width / 8); i += 256) {
        const int m = i / (width / 8), p = i % (width / 8);
        *reinterpret_cast<hg_bf16x8*>(y + (size_t)(m0 + m) * ys_t + (size_t)h * ys_h + c0 + p * 8) =
            *reinterpret_cast<const hg_bf16x8*>(ys + m * YP + p * 8);
      }
    } else {
      for (int i = threadIdx.x; i < here * width; i += 256) {
        const int m = i / width, p = i % width;
        y[(size_t)(m0 + m) * ys_t + (size_t)h * ys_h + c0 + p] = ys[m * YP + p];
      }
    }
    __syncthreads();
  }
}

extern "C" int nhv_head_gemm_bf16(const void* x, long long xs_t, long long xs_h, const void* w, void* y, long long ys_t,
                                  long long ys_h, const void* gate, int gate_mode, long long gs_t, int rows, int H, int N, int K,
                                  int rot, int x_rot_off, int y_rot_off, int halves, const void* freqs, float gain,
                                  const void* positions, void* stream) {
  NHV_REQUIRE(rows > 0 && H > 0 && H <= 65535 && N > 0 && K > 0, "head_gemm_bf16: bad sizes rows=%d H=%d N=%d K=%d", rows, H, N, K);
  NHV_REQUIRE(K % 8 == 0 && xs_t % 8 == 0 && xs_h % 8 == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)w % 16 == 0,
              "head_gemm_bf16: K=%d and the strides %lld, %lld must be multiples of 8, the operands 16 bytes aligned", K, xs_t, xs_h);
  NHV_REQUIRE(rot >= 0 && rot % 2 == 0 && (rot == 0 || (freqs != nullptr && positions != nullptr)),
              "head_gemm_bf16: a rotated part of %d entries needs frequencies and positions", rot);
  hipStream_t s = (hipStream_t)stream;
#define LAUNCH(MT, NT, WAVES, U)                                                                                          \
  do {                                                                                                                    \
    const int n_chunks = (N + 16 * NT * WAVES - 1) / (16 * NT * WAVES);                                                   \
    const dim3 grid(n_chunks + (rot > 0 ? 1 : 0), (rows + 16 * MT - 1) / (16 * MT), H);                                   \
    NHV_REQUIRE(grid.y <= 65535, "head_gemm_bf16: %d rows are too many", rows);                                           \
    hipLaunchKernelGGL((head_gemm_mfma_kernel<MT, NT, WAVES, U>), grid, dim3(64 * WAVES), 0, s, (const bf16_t*)x, xs_t, xs_h, \
                       (const bf16_t*)w, (bf16_t*)y, ys_t, ys_h, gate, gate_mode, gs_t, rows, N, K, n_chunks, rot,        \
                       x_rot_off, y_rot_off, halves, (const double*)freqs, gain, (const int*)positions);                  \
  } while (0)
  if (rows > 64 && K <= HT_MAX_K) {
    const size_t lds = (size_t)HT_ROWS * (K + 8 + HT_COLS + 8) * sizeof(bf16_t);
    auto kernel = head_gemm_tile_kernel<4>;
    // more than 64 KB of dynamic LDS has to be allowed once per kernel (and per process)
    static const hipError_t allowed = hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize,
                                                          (int)(HT_ROWS * (HT_MAX_K + 8 + HT_COLS + 8) * sizeof(bf16_t)));
    NHV_REQUIRE(allowed == hipSuccess, "head_gemm_bf16: %s", hipGetErrorString(allowed));
    const dim3 grid(H, (rows + HT_ROWS - 1) / HT_ROWS);
    NHV_REQUIRE(grid.y <= 65535, "head_gemm_bf16: %d rows are too many", rows);
    const int vec_out = N % 8 == 0 && ys_t % 8 == 0 && ys_h % 8 == 0 && (uintptr_t)y % 16 == 0;
    const int vec_gate = gate != nullptr && gate_mode == 2 && N % 4 == 0 && gs_t % 4 == 0 && (uintptr_t)gate % 8 == 0;
    hipLaunchKernelGGL(kernel, grid, dim3(256), lds, s, (const bf16_t*)x, xs_t, xs_h, (const bf16_t*)w, (bf16_t*)y, ys_t, ys_h, gate,
                       gate_mode, gs_t, rows, N, K, rot, x_rot_off, y_rot_off, halves, (const double*)freqs, gain,
                       (const int*)positions, vec_out, vec_gate);
  } else if (rows <= 16) {
    LAUNCH(1, 1, 1, 4);
  } else if (rows <= 64) {
    LAUNCH(2, 1, 4, 4);
  } else {
    LAUNCH(4, 2, 4, 2);
  }
#undef LAUNCH
  NHV_LAUNCH_CHECK("head_gemm_bf16");
  return 0;
}

// ---------------------------------------------------------------- the rotated part of the queries
// d[t, h, j] = turned s[t, h, j], j < rot; the rows of a (token, head) are s_t, s_h and d_t, d_h entries apart.
template <typename T>
__global__ void rotate_heads_kernel(const T* __restrict__ src, long long s_t, long long s_h, T* __restrict__ dst, long long d_t,
                                    long long d_h, int rot, int halves, const double* __restrict__ freqs, float gain,
                                    const int* __restrict__ positions, int H, size_t total) {
  const int half = rot / 2;
  for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (size_t)gridDim.x * blockDim.x) {
    const int p = (int)(i % half);
    const size_t t = i / half / H, h = i / half % H;
    nhv_turn_pair(src + t * s_t + h * s_h, dst + t * d_t + h * d_h, p, rot, halves, positions[t], freqs, gain);
  }
}

extern "C" int nhv_rotate_heads(const void* src, long long s_t, long long s_h, void* dst, long long d_t, long long d_h, int rot,
                                int halves, const void* freqs, float gain, const void* positions, int T, int H, int dtype,
                                void* stream) {
  NHV_REQUIRE(T > 0 && H > 0 && rot > 0 && rot % 2 == 0, "rotate_heads: bad sizes T=%d H=%d rot=%d", T, H, rot);
  NHV_REQUIRE(s_h >= rot && d_h >= rot && s_t >= s_h && d_t >= d_h, "rotate_heads: %d entries of rows %lld, %lld into %lld, %lld",
              rot, s_t, s_h, d_t, d_h);
  const size_t total = (size_t)T * H * (rot / 2);
  const int blocks = (int)((total + 255) / 256 > 65535 * 4 ? 65535 * 4 : (total + 255) / 256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == NHV_F32)
    hipLaunchKernelGGL(rotate_heads_kernel<float>, dim3(blocks), dim3(256), 0, s, (const float*)src, s_t, s_h, (float*)dst, d_t,
                       d_h, rot, halves, (const double*)freqs, gain, (const int*)positions, H, total);
  else if (dtype == NHV_BF16)
    hipLaunchKernelGGL(rotate_heads_kernel<bf16_t>, dim3(blocks), dim3(256), 0, s, (const bf16_t*)src, s_t, s_h, (bf16_t*)dst, d_t,
                       d_h, rot, halves, (const double*)freqs, gain, (const int*)positions, H, total);
  else
    return nhv_fail("rotate_heads: unknown dtype %d", dtype);
  NHV_LAUNCH_CHECK("rotate_heads");
  return 0;
}
