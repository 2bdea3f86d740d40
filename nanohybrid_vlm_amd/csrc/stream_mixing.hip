// Kernels around the residual stream and around attention for layers that are not the pre-norm kind:
//  - nhv_scalar_rmsnorm: RMS norm whose weight is one number;
//  - nhv_pair_norm_mean: half the sum of two rows, each RMS-normed with a weight vector of its own;
//  - nhv_depth_mix: a layer's result joins the list of all earlier results, and the stream that goes on is a
//    weighted sum over that list;
//  - nhv_rotary_split_write: splits a packed q | k | v projection whose value heads may have another size than
//    the key heads, adds biases, turns queries and keys (angles from the position and a list of frequencies,
//    taken in float here: no table, so no bound on positions) and optionally the values, scales queries by their
//    position, mixes values with another layer's, and stores keys and values at the step's slots.
// Statistics, angles and sums are float; rows are float or bfloat16.
#include "nhv_common.h"
#include "nhv_rotation.h"
#include <math.h>

// ---------------------------------------------------------------- norm with one number as its weight
template <typename TI, typename TO>
__global__ void scalar_rmsnorm_kernel(const TI* __restrict__ x, const float* __restrict__ gain, TO* __restrict__ y, int W,
                                      float eps) {
  __shared__ float scratch[16];
  const size_t base = (size_t)blockIdx.x * W;
  float ss = 0.f;
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    const float v = to_f32(x[base + i]);
    ss = fmaf(v, v, ss);
  }
  const float total = block_sum(ss, scratch);
  const float r = gain[0] / sqrtf(total / (float)W + eps);
  for (int i = threadIdx.x; i < W; i += blockDim.x) y[base + i] = from_f32<TO>(to_f32(x[base + i]) * r);
}

extern "C" int nhv_scalar_rmsnorm(const void* x, int x_dtype, const void* gain, void* y, int y_dtype, int T, int W, float eps,
                                  void* stream) {
  NHV_REQUIRE(T > 0 && W > 0, "scalar_rmsnorm: bad sizes T=%d W=%d", T, W);
  hipStream_t s = (hipStream_t)stream;
#define LAUNCH(TI, TO)                                                                                               \
  hipLaunchKernelGGL((scalar_rmsnorm_kernel<TI, TO>), dim3(T), dim3(256), 0, s, (const TI*)x, (const float*)gain, (TO*)y, \
                     W, eps)
  if (x_dtype == NHV_F32 && y_dtype == NHV_F32) LAUNCH(float, float);
  else if (x_dtype == NHV_F32 && y_dtype == NHV_BF16) LAUNCH(float, bf16_t);
  else if (x_dtype == NHV_BF16 && y_dtype == NHV_F32) LAUNCH(bf16_t, float);
  else if (x_dtype == NHV_BF16 && y_dtype == NHV_BF16) LAUNCH(bf16_t, bf16_t);
  else return nhv_fail("scalar_rmsnorm: unknown dtypes %d -> %d", x_dtype, y_dtype);
#undef LAUNCH
  NHV_LAUNCH_CHECK("scalar_rmsnorm");
  return 0;
}

// ---------------------------------------------------------------- two normed rows, half their sum
template <typename T>
__global__ void pair_norm_mean_kernel(const T* __restrict__ a, const float* __restrict__ wa, const T* __restrict__ b,
                                      const float* __restrict__ wb, T* __restrict__ y, int W, float eps) {
  __shared__ float scratch[16];
  const size_t base = (size_t)blockIdx.x * W;
  float sa = 0.f, sb = 0.f;
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    const float u = to_f32(a[base + i]), v = to_f32(b[base + i]);
    sa = fmaf(u, u, sa);
    sb = fmaf(v, v, sb);
  }
  const float ra = 1.0f / sqrtf(block_sum(sa, scratch) / (float)W + eps);
  const float rb = 1.0f / sqrtf(block_sum(sb, scratch) / (float)W + eps);
  for (int i = threadIdx.x; i < W; i += blockDim.x)
    y[base + i] = from_f32<T>(0.5f * (to_f32(a[base + i]) * ra * wa[i] + to_f32(b[base + i]) * rb * wb[i]));
}

extern "C" int nhv_pair_norm_mean(const void* a, const void* wa, const void* b, const void* wb, void* y, int T, int W,
                                  float eps, int dtype, void* stream) {
  NHV_REQUIRE(T > 0 && W > 0, "pair_norm_mean: bad sizes T=%d W=%d", T, W);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == NHV_F32)
    hipLaunchKernelGGL(pair_norm_mean_kernel<float>, dim3(T), dim3(256), 0, s, (const float*)a, (const float*)wa,
                       (const float*)b, (const float*)wb, (float*)y, W, eps);
  else if (dtype == NHV_BF16)
    hipLaunchKernelGGL(pair_norm_mean_kernel<bf16_t>, dim3(T), dim3(256), 0, s, (const bf16_t*)a, (const float*)wa,
                       (const bf16_t*)b, (const float*)wb, (bf16_t*)y, W, eps);
  else return nhv_fail("pair_norm_mean: unknown dtype %d", dtype);
  NHV_LAUNCH_CHECK("pair_norm_mean");
  return 0;
}

// ---------------------------------------------------------------- weighted sum over all results so far
// results[0 .. n) are [rows, W] float each, n = index + 2. results[index + 1] = x + (a + b) is written here (and
// results[0] = x when index is 0: the stream that enters the first layer is the first result); then
// out = sum over j < n of weights[j] * results[j], in rising j. With ``gain`` the RMS norm of out with that one number
// as its weight is written to ``normed`` as well (what the next layer reads). With ``a2`` the first addend is not a but
// half the sum of a and a2, each over its root mean square (pair_eps) times its weight vector wa, wb: what
// nhv_pair_norm_mean would have written, unrounded.
template <typename T>
__global__ void depth_mix_kernel(const float* __restrict__ x, const T* __restrict__ a, const T* __restrict__ b,
                                 float* __restrict__ results, size_t plane, int index, const float* __restrict__ weights,
                                 float* __restrict__ out, const float* __restrict__ gain, T* __restrict__ normed, int W,
                                 float eps, const T* __restrict__ a2, const float* __restrict__ wa,
                                 const float* __restrict__ wb, float pair_eps) {
  __shared__ float scratch[16];
  const size_t base = (size_t)blockIdx.x * W;
  const int n = index + 2;
  float ra = 1.f, rb = 0.f;
  if (a2 != nullptr) {
    float sa = 0.f, sb = 0.f;
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
      const float u = to_f32(a[base + i]), v = to_f32(a2[base + i]);
      sa = fmaf(u, u, sa);
      sb = fmaf(v, v, sb);
    }
    ra = 1.0f / sqrtf(block_sum(sa, scratch) / (float)W + pair_eps);
    rb = 1.0f / sqrtf(block_sum(sb, scratch) / (float)W + pair_eps);
  }
  float ss = 0.f;
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    const float xi = x[base + i];
    float add = a2 != nullptr ? 0.5f * (to_f32(a[base + i]) * ra * wa[i] + to_f32(a2[base + i]) * rb * wb[i]) : to_f32(a[base + i]);
    if (b != nullptr) add += to_f32(b[base + i]);
    const float mine = xi + add;
    results[(size_t)(index + 1) * plane + base + i] = mine;
    if (index == 0) results[base + i] = xi;
    float sum = 0.f;
    for (int j = 0; j + 1 < n; ++j) sum = fmaf(weights[j], j == 0 && index == 0 ? xi : results[(size_t)j * plane + base + i], sum);
    sum = fmaf(weights[n - 1], mine, sum);
    out[base + i] = sum;
    ss = fmaf(sum, sum, ss);
  }
  if (gain == nullptr) return;
  const float total = block_sum(ss, scratch);
  const float r = gain[0] / sqrtf(total / (float)W + eps);
  for (int i = threadIdx.x; i < W; i += blockDim.x) normed[base + i] = from_f32<T>(out[base + i] * r);
}

extern "C" int nhv_depth_mix(const void* x, const void* a, const void* b, void* results, long long plane, int index,
                             const void* weights, void* out, const void* gain, void* normed, int T, int W, float eps,
                             const void* a2, const void* wa, const void* wb, float pair_eps, int dtype, void* stream) {
  NHV_REQUIRE(T > 0 && W > 0 && index >= 0 && plane >= (long long)T * W, "depth_mix: bad sizes T=%d W=%d index=%d", T, W, index);
  NHV_REQUIRE(x != out, "depth_mix: the sum cannot be written over the stream it reads");
  NHV_REQUIRE(a2 == nullptr || (wa != nullptr && wb != nullptr), "depth_mix: a pair of addends without its weights");
  hipStream_t s = (hipStream_t)stream;
  if (dtype == NHV_F32)
    hipLaunchKernelGGL(depth_mix_kernel<float>, dim3(T), dim3(256), 0, s, (const float*)x, (const float*)a, (const float*)b,
                       (float*)results, (size_t)plane, index, (const float*)weights, (float*)out, (const float*)gain,
                       (float*)normed, W, eps, (const float*)a2, (const float*)wa, (const float*)wb, pair_eps);
  else if (dtype == NHV_BF16)
    hipLaunchKernelGGL(depth_mix_kernel<bf16_t>, dim3(T), dim3(256), 0, s, (const float*)x, (const bf16_t*)a, (const bf16_t*)b,
                       (float*)results, (size_t)plane, index, (const float*)weights, (float*)out, (const float*)gain,
                       (bf16_t*)normed, W, eps, (const bf16_t*)a2, (const float*)wa, (const float*)wb, pair_eps);
  else return nhv_fail("depth_mix: unknown dtype %d", dtype);
  NHV_LAUNCH_CHECK("depth_mix");
  return 0;
}

// ---------------------------------------------------------------- split, bias, rotation, store
// qkv [T, ld]: q (Hq heads of D) | k (Hkv heads of D) | v (Hv heads of E) | further columns of another reader; one wave
// per (token, head). A query or key head at position p turns over its first ``rot`` coordinates by p * qk_freqs[i]:
// pair (i, i + rot / 2), or (2i, 2i + 1) where ``interleaved``; the coordinates from rot on pass. v_freqs [E / 2] or
// null: pair (m, m + E / 2) of a value head turns by p * v_freqs[m]. ``unit``: after the rotation every query and key
// head is divided by its root mean square (unit_eps under the root), in float before anything is rounded.
// ``v_from_k``: there are no value columns; value head g is key head g as projected (bias added, not turned, not
// normed). ``maps`` n > 1: every query and key head holds n maps of D entries, [map 1 | map 2 | ...], each turned (and
// normed) on its own; Hq and Hkv count maps. The n maps of a key head are stored side by side as one key of n D entries
// (there are Hkv / n key heads, and as many value heads); a query map goes out as a head of n D entries of its own
// with zeros in the other maps' places, so that its product with the stored key is its product with its own map.
// ``q_every`` > 0: queries at position p are multiplied by 1 + q_coef ln(floor((p + 1) / q_every) + 1). ``v_first``: value
// head g becomes (1 - lam) v + lam v1, v1 the entries of value head g at v_first[t * v_first_ld + g E ...] (rows of
// another layer's projection, of the same token), lam the number at v_lam; all in float, rounded once.
struct SplitMore {
  float q_coef;
  double q_every;
  const void* v_first;
  long long v_first_ld;
  const float* v_lam;
};

__device__ __forceinline__ float query_temperature(int pos, const SplitMore& more) {
  if (!(more.q_every > 0.0)) return 1.0f;
  return 1.0f + more.q_coef * logf((float)floor(((double)pos + 1.0) / more.q_every) + 1.0f);
}

template <typename T>
__global__ void rotary_split_write_kernel(const T* __restrict__ qkv, const T* __restrict__ bias,
                                          const float* __restrict__ qk_freqs, int rot, const float* __restrict__ v_freqs,
                                          const int* __restrict__ positions, const int* __restrict__ slot_mapping,
                                          T* __restrict__ q_out, T* __restrict__ k_cache, T* __restrict__ v_cache, int Hq,
                                          int Hkv, int Hv, int D, int E, int heads, int ld, int interleaved, int unit,
                                          float unit_eps, int v_from_k, int maps, const SplitMore more) {
  extern __shared__ float staged[];            // D floats where heads are normed: the head after bias and rotation
  const int t = blockIdx.x / heads, head = blockIdx.x % heads;
  const float p = (float)positions[t];
  int col, size, half;
  bool normed = false, pairs_adjacent = false;
  const float* freqs;
  T* dst;
  const T* first = nullptr;                    // what a value head is mixed with, by lam
  float factor = 1.0f, lam = 0.0f;
  if (head < Hq) {
    factor = query_temperature(positions[t], more);
    col = head * D; size = D; half = rot / 2; freqs = qk_freqs; normed = unit; pairs_adjacent = interleaved;
    T* whole = q_out + ((size_t)t * Hq + head) * maps * D;
    dst = whole + (head % maps) * D;
    if (maps > 1)                              // the other maps' places
      for (int i = threadIdx.x; i < maps * D; i += blockDim.x)
        if (i / D != head % maps) whole[i] = from_f32<T>(0.f);
  } else {
    const int slot = slot_mapping[t];
    if (slot < 0) return;                      // a row that stores nothing (padding of a recorded step)
    if (head < Hq + Hkv) {
      const int g = head - Hq;
      col = Hq * D + g * D; size = D; half = rot / 2; freqs = qk_freqs; normed = unit; pairs_adjacent = interleaved;
      dst = k_cache + ((size_t)slot * Hkv + g) * D;          // (map g % maps of key head g / maps: the same place)
    } else {
      const int g = head - Hq - Hkv;
      col = v_from_k ? Hq * D + g * D : (Hq + Hkv) * D + g * E;
      size = E; half = v_freqs ? E / 2 : 0; freqs = v_freqs;
      dst = v_cache + ((size_t)slot * Hv + g) * E;
      if (more.v_first) {
        first = reinterpret_cast<const T*>(more.v_first) + (size_t)t * more.v_first_ld + g * E;
        lam = *more.v_lam;
      }
    }
  }
  const T* src = qkv + (size_t)t * ld + col;
  const T* bs = bias ? bias + col : nullptr;
  // the bias joins a projection that was rounded to the rows' type, and the sum is rounded again (the product's own result)
  auto value = [&](int i) {
    float v = bs ? to_f32(from_f32<T>(to_f32(src[i]) + to_f32(bs[i]))) : to_f32(src[i]);
    if (first) v = (1.0f - lam) * v + lam * to_f32(first[i]);
    return v;
  };
  if (!normed) {                               // nothing of the head depends on all of it: every entry goes out at once
    for (int i = threadIdx.x; i < size - half; i += blockDim.x) {
      if (i < half) {
        const int a = pairs_adjacent ? 2 * i : i, b = pairs_adjacent ? 2 * i + 1 : i + half;
        const float u = value(a), v = value(b);
        float sn, cs;
        sincosf(p * freqs[i], &sn, &cs);
        dst[a] = from_f32<T>((u * cs - v * sn) * factor);
        dst[b] = from_f32<T>((v * cs + u * sn) * factor);
      } else {
        dst[i + half] = from_f32<T>(value(i + half) * factor);
      }
    }
    return;
  }
  // the unit norm follows the rotation: the turned head waits in LDS as floats for its sum of squares
  float ss = 0.f;
  for (int i = threadIdx.x; i < size - half; i += blockDim.x) {
    if (i < half) {
      const int a = pairs_adjacent ? 2 * i : i, b = pairs_adjacent ? 2 * i + 1 : i + half;
      const float u = value(a), v = value(b);
      float sn, cs;
      sincosf(p * freqs[i], &sn, &cs);
      const float x = u * cs - v * sn, y = v * cs + u * sn;
      staged[a] = x;
      staged[b] = y;
      ss = fmaf(x, x, fmaf(y, y, ss));
    } else {
      const float x = value(i + half);
      staged[i + half] = x;
      ss = fmaf(x, x, ss);
    }
  }
  const float r = factor / sqrtf(wave_sum(ss) / (float)size + unit_eps);
  __syncthreads();
  for (int i = threadIdx.x; i < size; i += blockDim.x) dst[i] = from_f32<T>(staged[i] * r);
}

// The same where nothing is turned or normed and heads are whole pieces of eight entries: a thread moves eight entries of
// one row (16 bytes in bfloat16), whatever head they belong to. blockIdx.x walks along the row, blockIdx.y over tokens.
template <typename T>
__device__ __forceinline__ void split_load8(const T* p, float* v) {
  struct alignas(sizeof(T) * 8) Pack { T e[8]; };
  const Pack pack = *reinterpret_cast<const Pack*>(p);
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = to_f32(pack.e[i]);
}

template <typename T>
__global__ __launch_bounds__(256) void split_write_vec_kernel(const T* __restrict__ qkv, const int* __restrict__ positions,
                                                              const int* __restrict__ slot_mapping, T* __restrict__ q_out,
                                                              T* __restrict__ k_cache, T* __restrict__ v_cache, int nq, int nk,
                                                              int nv, int ld, int T_rows, const SplitMore more) {
  struct alignas(sizeof(T) * 8) Pack { T e[8]; };
  const int c = (blockIdx.x * 256 + threadIdx.x) * 8;
  if (c >= nq + nk + nv) return;
  for (int t = blockIdx.y; t < T_rows; t += gridDim.y) {
    Pack in = *reinterpret_cast<const Pack*>(qkv + (size_t)t * ld + c);
    if (c < nq) {
      const float factor = query_temperature(positions[t], more);
      if (factor != 1.0f)
#pragma unroll
        for (int i = 0; i < 8; ++i) in.e[i] = from_f32<T>(to_f32(in.e[i]) * factor);
      *reinterpret_cast<Pack*>(q_out + (size_t)t * nq + c) = in;
      continue;
    }
    const int slot = slot_mapping[t];
    if (slot < 0) continue;                    // a row that stores nothing (padding of a recorded step)
    if (c < nq + nk) {
      *reinterpret_cast<Pack*>(k_cache + (size_t)slot * nk + (c - nq)) = in;
      continue;
    }
    const int at = c - nq - nk;
    if (more.v_first) {
      float first[8];
      split_load8(reinterpret_cast<const T*>(more.v_first) + (size_t)t * more.v_first_ld + at, first);
      const float lam = *more.v_lam;
#pragma unroll
      for (int i = 0; i < 8; ++i) in.e[i] = from_f32<T>((1.0f - lam) * to_f32(in.e[i]) + lam * first[i]);
    }
    *reinterpret_cast<Pack*>(v_cache + (size_t)slot * nv + at) = in;
  }
}

extern "C" int nhv_rotary_split_write(const void* qkv, const void* bias, const void* qk_freqs, int rot, const void* v_freqs,
                                      const void* positions, const void* slot_mapping, void* q_out, void* k_cache,
                                      void* v_cache, int T, int Hq, int Hkv, int D, int E, int with_kv, int more_columns,
                                      int interleaved, int unit, float unit_eps, int v_from_k, int maps, float q_coef,
                                      double q_every, const void* v_first, long long v_first_ld, const void* v_lam, int dtype,
                                      void* stream) {
  NHV_REQUIRE(more_columns >= 0, "rotary_split_write: %d columns after the projection", more_columns);
  NHV_REQUIRE(T > 0 && Hq > 0 && Hkv > 0 && D > 0 && E > 0, "rotary_split_write: bad sizes T=%d Hq=%d Hkv=%d D=%d E=%d", T, Hq, Hkv, D, E);
  NHV_REQUIRE(rot >= 0 && rot % 2 == 0 && rot <= D, "rotary_split_write: rotary size %d with head size %d", rot, D);
  NHV_REQUIRE(rot == 0 || qk_freqs, "rotary_split_write: a rotary size without frequencies");
  NHV_REQUIRE(!v_freqs || E % 2 == 0, "rotary_split_write: value heads of odd size %d cannot be turned", E);
  NHV_REQUIRE(!with_kv || (slot_mapping && k_cache && v_cache), "rotary_split_write: cache write without cache");
  NHV_REQUIRE(maps >= 1 && Hq % maps == 0 && Hkv % maps == 0, "rotary_split_write: %d maps with %d and %d heads", maps, Hq, Hkv);
  NHV_REQUIRE(!v_from_k || (E == D && maps == 1), "rotary_split_write: values that are the keys as projected have the keys' size and one map");
  NHV_REQUIRE(!unit || unit_eps >= 0.f, "rotary_split_write: eps %g", (double)unit_eps);
  const int Hv = Hkv / maps;
  NHV_REQUIRE(!v_first || (with_kv && v_lam && !v_freqs && v_first_ld >= (long long)Hv * E),
              "rotary_split_write: values mixed with others need both, unturned, and rows of at least %d entries (%lld)", Hv * E, v_first_ld);
  NHV_REQUIRE(q_every >= 0.0, "rotary_split_write: queries scaled in steps of %g positions", q_every);
  const SplitMore more = {q_coef, q_every, v_first, v_first_ld, (const float*)v_lam};
  const int heads = with_kv ? Hq + Hkv + Hv : Hq;
  const int ld = (with_kv ? Hq * D + Hkv * D + (v_from_k ? 0 : Hv * E) : Hq * D) + more_columns;   // (columns that belong to another reader)
  NHV_REQUIRE((long long)T * heads < (1ll << 31), "rotary_split_write: too many tokens");
  const size_t item = dtype == NHV_F32 ? 4 : 2;
  const uintptr_t starts = (uintptr_t)qkv | (uintptr_t)q_out | (uintptr_t)k_cache | (uintptr_t)v_cache | (uintptr_t)v_first;
  if (with_kv && rot == 0 && !unit && !v_freqs && !bias && !v_from_k && maps == 1 && D % 8 == 0 && E % 8 == 0 && ld % 8 == 0 &&
      v_first_ld % 8 == 0 && starts % (8 * item) == 0 && (dtype == NHV_F32 || dtype == NHV_BF16)) {
    const int nq = Hq * D, nk = Hkv * D, nv = Hkv * E;
    const dim3 grid(((nq + nk + nv) / 8 + 255) / 256, T < 65535 ? T : 65535);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == NHV_F32)
      hipLaunchKernelGGL(split_write_vec_kernel<float>, grid, dim3(256), 0, s, (const float*)qkv, (const int*)positions,
                         (const int*)slot_mapping, (float*)q_out, (float*)k_cache, (float*)v_cache, nq, nk, nv, ld, T, more);
    else
      hipLaunchKernelGGL(split_write_vec_kernel<bf16_t>, grid, dim3(256), 0, s, (const bf16_t*)qkv, (const int*)positions,
                         (const int*)slot_mapping, (bf16_t*)q_out, (bf16_t*)k_cache, (bf16_t*)v_cache, nq, nk, nv, ld, T, more);
    NHV_LAUNCH_CHECK("split_write_vec");
    return 0;
  }
  const size_t lds = unit ? (size_t)D * sizeof(float) : 0;
  NHV_REQUIRE(lds <= 64 * 1024, "rotary_split_write: heads of %d entries are beyond this kernel's unit norm", D);
  hipStream_t s = (hipStream_t)stream;
#define LAUNCH(TT)                                                                                                   \
  hipLaunchKernelGGL(rotary_split_write_kernel<TT>, dim3((unsigned)((size_t)T * heads)), dim3(NHV_WAVE), lds, s,     \
                     (const TT*)qkv, (const TT*)bias, (const float*)qk_freqs, rot, (const float*)v_freqs,            \
                     (const int*)positions, (const int*)slot_mapping, (TT*)q_out, (TT*)k_cache, (TT*)v_cache, Hq, Hkv, Hv, \
                     D, E, heads, ld, interleaved, unit, unit_eps, v_from_k, maps, more)
  if (dtype == NHV_F32) LAUNCH(float);
  else if (dtype == NHV_BF16) LAUNCH(bf16_t);
  else return nhv_fail("rotary_split_write: unknown dtype %d", dtype);
#undef LAUNCH
  NHV_LAUNCH_CHECK("rotary_split_write");
  return 0;
}

// ---------------------------------------------------------------- queries and keys normed over their whole projection
// Packed rows q (Hq D) | k (Hkv D) | v (Hkv E, absent where the values are the keys as projected), plus bias. All of q is
// divided by its root mean square and multiplied by wq entry by entry, all of k likewise by wk; then pairs (i, i + rot / 2) of every head
// turn by position * freqs[i] (doubles), cosine and sine times gain; q goes to q_out, keys and values to the step's slots. One
// block a token: the sums of squares meet in LDS, and so do the token's sines and cosines, which all heads share.
template <typename T>
__global__ __launch_bounds__(256) void normed_split_write_kernel(const T* __restrict__ qkv, int ld, const T* __restrict__ bias,
                                                                 const float* __restrict__ wq, const float* __restrict__ wk,
                                                                 float eps, const double* __restrict__ freqs, int rot, float gain,
                                                                 const int* __restrict__ positions,
                                                                 const int* __restrict__ slot_mapping, T* __restrict__ q_out,
                                                                 T* __restrict__ k_cache, T* __restrict__ v_cache, int Hq, int Hkv,
                                                                 int D, int E, int v_from_k) {
  extern __shared__ float turns[];             // rot / 2 sines, then as many cosines
  __shared__ float scratch[16];
  const int t = blockIdx.x, nq = Hq * D, nk = Hkv * D, half = rot / 2;
  const T* row = qkv + (size_t)t * ld;
  auto value = [&](int c) { return bias ? to_f32(row[c]) + to_f32(bias[c]) : to_f32(row[c]); };
  for (int i = threadIdx.x; i < half; i += 256) nhv_turn_angle<float>(positions[t], freqs[i], gain, &turns[i], &turns[half + i]);
  float sq = 0.f, sk = 0.f;
  for (int c = threadIdx.x; c < nq; c += 256) {
    const float v = value(c);
    sq = fmaf(v, v, sq);
  }
  for (int c = nq + threadIdx.x; c < nq + nk; c += 256) {
    const float v = value(c);
    sk = fmaf(v, v, sk);
  }
  const float rq = 1.0f / sqrtf(block_sum(sq, scratch) / (float)nq + eps);
  const float rk = 1.0f / sqrtf(block_sum(sk, scratch) / (float)nk + eps);    // (its barriers show the sines as well)
  const int slot = slot_mapping[t];
  const int per = D - half;                    // pairs, then what is not turned
  const int heads = slot < 0 ? Hq : Hq + Hkv;  // (a row that stores nothing: padding of a recorded step)
  for (int x = threadIdx.x; x < heads * per; x += 256) {
    const int h = x / per, i = x % per;
    const bool key = h >= Hq;
    const float* w = key ? wk + (size_t)(h - Hq) * D : wq + (size_t)h * D;
    const float r = key ? rk : rq;
    T* dst = key ? k_cache + ((size_t)slot * Hkv + h - Hq) * D : q_out + ((size_t)t * Hq + h) * D;
    const int c = h * D;
    if (i < half) {
      const float a = value(c + i), b = value(c + i + half);
      const float u = a * r * w[i], v = b * r * w[i + half];
      dst[i] = from_f32<T>(u * turns[half + i] - v * turns[i]);
      dst[i + half] = from_f32<T>(v * turns[half + i] + u * turns[i]);
      if (key && v_from_k) {
        T* vd = v_cache + ((size_t)slot * Hkv + h - Hq) * E;
        vd[i] = from_f32<T>(a);
        vd[i + half] = from_f32<T>(b);
      }
    } else {
      const float a = value(c + i + half);
      dst[i + half] = from_f32<T>(a * r * w[i + half]);
      if (key && v_from_k) v_cache[((size_t)slot * Hkv + h - Hq) * E + i + half] = from_f32<T>(a);
    }
  }
  if (slot >= 0 && !v_from_k)
    for (int c = threadIdx.x; c < Hkv * E; c += 256) v_cache[(size_t)slot * Hkv * E + c] = from_f32<T>(value(nq + nk + c));
}

// The same where heads and halves are whole pieces of eight entries: a thread moves eight entries at a time, the row waits in
// LDS as floats for its sums of squares (a pair's two entries lie in different threads' pieces).
template <typename T>
__global__ __launch_bounds__(1024) void normed_split_write_vec_kernel(const T* __restrict__ qkv, int ld, const T* __restrict__ bias,
                                                                      const float* __restrict__ wq, const float* __restrict__ wk,
                                                                      float eps, const double* __restrict__ freqs, int rot,
                                                                      float gain, const int* __restrict__ positions,
                                                                      const int* __restrict__ slot_mapping, T* __restrict__ q_out,
                                                                      T* __restrict__ k_cache, T* __restrict__ v_cache, int nq,
                                                                      int nk, int nv, int D, int v_from_k) {
  struct alignas(sizeof(T) * 8) Pack { T e[8]; };
  extern __shared__ __attribute__((aligned(16))) float row_s[];      // nq + nk values, then rot / 2 sines and as many cosines
  __shared__ float scratch[16];
  const int t = blockIdx.x, half = rot / 2, n = nq + nk, threads = blockDim.x;
  float* sines = row_s + n;
  float* cosines = sines + half;
  const T* row = qkv + (size_t)t * ld;
  const int slot = slot_mapping[t];
  float sq = 0.f, sk = 0.f;
  for (int c = threadIdx.x * 8; c < n + nv; c += threads * 8) {
    float v[8];
    split_load8(row + c, v);
    if (bias) {
      float b[8];
      split_load8(bias + c, b);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] += b[i];
    }
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) ss = fmaf(v[i], v[i], ss);
    if (c < nq) sq += ss;
    else if (c < n) sk += ss;
    if (c < n) {
      *reinterpret_cast<float4*>(row_s + c) = float4{v[0], v[1], v[2], v[3]};
      *reinterpret_cast<float4*>(row_s + c + 4) = float4{v[4], v[5], v[6], v[7]};
    }
    if (slot >= 0 && (v_from_k ? (c >= nq && c < n) : c >= n)) {     // (a row that stores nothing: padding of a recorded step)
      Pack out;
#pragma unroll
      for (int i = 0; i < 8; ++i) out.e[i] = from_f32<T>(v[i]);
      *reinterpret_cast<Pack*>(v_cache + (v_from_k ? (size_t)slot * nk + (c - nq) : (size_t)slot * nv + (c - n))) = out;
    }
  }
  for (int i = threadIdx.x; i < half; i += threads) nhv_turn_angle<float>(positions[t], freqs[i], gain, &sines[i], &cosines[i]);
  const float rq = 1.0f / sqrtf(block_sum(sq, scratch) / (float)nq + eps);
  const float rk = 1.0f / sqrtf(block_sum(sk, scratch) / (float)nk + eps);    // (its barriers show the row and the sines as well)
  for (int c = threadIdx.x * 8; c < (slot < 0 ? nq : n); c += threads * 8) {
    const bool key = c >= nq;
    const int in_head = c % D;
    const float* w = key ? wk + (c - nq) : wq + c;
    const float r = key ? rk : rq;
    const int other = in_head < half ? half : -half;                 // where the pairs' other entries lie
    float v[8], wv[8];
    split_load8(row_s + c, v);
    split_load8(w, wv);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= r * wv[i];
    if (in_head < rot) {
      float x[8], sn[8], cs[8];
      split_load8(row_s + c + other, x);
      split_load8(w + other, wv);
      const int p = in_head < half ? in_head : in_head - half;
      split_load8(sines + p, sn);
      split_load8(cosines + p, cs);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float y = x[i] * r * wv[i];
        v[i] = in_head < half ? v[i] * cs[i] - y * sn[i] : v[i] * cs[i] + y * sn[i];
      }
    }
    Pack out;
#pragma unroll
    for (int i = 0; i < 8; ++i) out.e[i] = from_f32<T>(v[i]);
    *reinterpret_cast<Pack*>(key ? k_cache + (size_t)slot * nk + (c - nq) : q_out + (size_t)t * nq + c) = out;
  }
}

extern "C" int nhv_normed_split_write(const void* qkv, long long ld, const void* bias, const void* wq, const void* wk, float eps,
                                      const void* freqs, int rot, float gain, const void* positions, const void* slot_mapping,
                                      void* q_out, void* k_cache, void* v_cache, int T, int Hq, int Hkv, int D, int E,
                                      int v_from_k, int dtype, void* stream) {
  NHV_REQUIRE(T > 0 && Hq > 0 && Hkv > 0 && D > 0 && E > 0, "normed_split_write: bad sizes T=%d Hq=%d Hkv=%d D=%d E=%d", T, Hq, Hkv, D, E);
  NHV_REQUIRE(rot >= 0 && rot % 2 == 0 && rot <= D && (rot == 0 || freqs) && rot <= 8192, "normed_split_write: rotary size %d with head size %d", rot, D);
  NHV_REQUIRE(!v_from_k || E == D, "normed_split_write: values that are the keys as projected have the keys' size");
  NHV_REQUIRE(ld >= (long long)(Hq + Hkv) * D + (v_from_k ? 0 : Hkv * E) && ld < (1ll << 31), "normed_split_write: rows of %lld entries", ld);
  NHV_REQUIRE(wq && wk && slot_mapping && k_cache && v_cache && eps >= 0.f, "normed_split_write: norm weights, slots and caches are needed");
  hipStream_t s = (hipStream_t)stream;
  const size_t item = dtype == NHV_F32 ? 4 : 2;
  const uintptr_t starts = (uintptr_t)qkv | (uintptr_t)bias | (uintptr_t)q_out | (uintptr_t)k_cache | (uintptr_t)v_cache;
  const uintptr_t w_starts = (uintptr_t)wq | (uintptr_t)wk;
  const int nq = Hq * D, nk = Hkv * D, nv = v_from_k ? 0 : Hkv * E;
  const size_t row_lds = ((size_t)nq + nk + rot) * sizeof(float);
  if (D % 8 == 0 && rot % 16 == 0 && (v_from_k || E % 8 == 0) && ld % 8 == 0 && starts % (8 * item) == 0 && w_starts % 32 == 0 &&
      row_lds <= 60 * 1024 &&
      (dtype == NHV_F32 || dtype == NHV_BF16)) {
    int threads = ((nq + nk + nv) / 8 + 63) / 64 * 64;
    if (threads > 1024) threads = 1024;
#define LAUNCH_VEC(TT)                                                                                                    \
  hipLaunchKernelGGL(normed_split_write_vec_kernel<TT>, dim3(T), dim3(threads), row_lds, s, (const TT*)qkv, (int)ld,      \
                     (const TT*)bias, (const float*)wq, (const float*)wk, eps, (const double*)freqs, rot, gain,           \
                     (const int*)positions, (const int*)slot_mapping, (TT*)q_out, (TT*)k_cache, (TT*)v_cache, nq, nk, nv, D, v_from_k)
    if (dtype == NHV_F32) LAUNCH_VEC(float);
    else LAUNCH_VEC(bf16_t);
#undef LAUNCH_VEC
    NHV_LAUNCH_CHECK("normed_split_write_vec");
    return 0;
  }
#define LAUNCH(TT)                                                                                                        \
  hipLaunchKernelGGL(normed_split_write_kernel<TT>, dim3(T), dim3(256), (size_t)rot * sizeof(float), s, (const TT*)qkv, (int)ld, \
                     (const TT*)bias, (const float*)wq, (const float*)wk, eps, (const double*)freqs, rot, gain,           \
                     (const int*)positions, (const int*)slot_mapping, (TT*)q_out, (TT*)k_cache, (TT*)v_cache, Hq, Hkv, D, E, \
                     v_from_k)
  if (dtype == NHV_F32) LAUNCH(float);
  else if (dtype == NHV_BF16) LAUNCH(bf16_t);
  else return nhv_fail("normed_split_write: unknown dtype %d", dtype);
#undef LAUNCH
  NHV_LAUNCH_CHECK("normed_split_write");
  return 0;
}

// ---------------------------------------------------------------- heads turned back by their position
// x[T, H, E] in place: pair (m, m + E / 2) of every head at position p turns by -p * freqs[m].
template <typename T>
__global__ void turn_back_kernel(T* __restrict__ x, const float* __restrict__ freqs, const int* __restrict__ positions, int H,
                                 int E) {
  const int t = blockIdx.x / H;
  const float p = (float)positions[t];
  T* row = x + (size_t)blockIdx.x * E;
  const int half = E / 2;
  for (int m = threadIdx.x; m < half; m += blockDim.x) {
    const float u = to_f32(row[m]), v = to_f32(row[m + half]);
    float sn, cs;
    sincosf(p * freqs[m], &sn, &cs);
    row[m] = from_f32<T>(u * cs + v * sn);
    row[m + half] = from_f32<T>(v * cs - u * sn);
  }
}

extern "C" int nhv_turn_back(void* x, const void* freqs, const void* positions, int T, int H, int E, int dtype, void* stream) {
  NHV_REQUIRE(T > 0 && H > 0 && E > 0 && E % 2 == 0, "turn_back: bad sizes T=%d H=%d E=%d", T, H, E);
  NHV_REQUIRE((long long)T * H < (1ll << 31), "turn_back: too many tokens");
  hipStream_t s = (hipStream_t)stream;
  if (dtype == NHV_F32)
    hipLaunchKernelGGL(turn_back_kernel<float>, dim3((unsigned)((size_t)T * H)), dim3(NHV_WAVE), 0, s, (float*)x,
                       (const float*)freqs, (const int*)positions, H, E);
  else if (dtype == NHV_BF16)
    hipLaunchKernelGGL(turn_back_kernel<bf16_t>, dim3((unsigned)((size_t)T * H)), dim3(NHV_WAVE), 0, s, (bf16_t*)x,
                       (const float*)freqs, (const int*)positions, H, E);
  else return nhv_fail("turn_back: unknown dtype %d", dtype);
  NHV_LAUNCH_CHECK("turn_back");
  return 0;
}
