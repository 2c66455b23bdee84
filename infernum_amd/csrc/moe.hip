// Routed experts: a token's feed-forward is the weighted sum of `top` small gated feed-forwards chosen among E.
//   ia_router_topk   z = logits + bias (fp32); the `top` largest (the lowest index among equals) and the softmax
//                    over those alone;
//   ia_moe_sort      the (token, choice) pairs grouped by expert: offsets[E + 1], perm[P];
//   ia_moe_gate_up   per expert, over its pairs' tokens: g = min(Wg x, limit), u = clamp(Wu x, -limit, limit),
//                    y = g sigmoid(alpha g) (u + shift); the rows of Wg and Wu alternate in the expert's matrix (limit
//                    infinity, alpha 1, shift 0: y = silu(Wg x) (Wu x));
//   ia_moe_down      per expert: Wd y times the pair's routing weight, as fp32 into parts[choice, token, :], which
//                    the kernel that takes the feed-forward's result next adds in the order of the choices.
// A routing weight can stand on the expert's INPUT instead: ia_moe_gate_up (and ia_moe_glu) given the weights multiply
// both products with it, in fp32 (G (w x) = w (G x)), and ia_moe_down (and ia_moe_scatter) given none leave theirs as it is.
// Only the chosen experts' weights are read.  A pair's result is one chain of operations over its own token and
// its expert's weights, whatever else the step holds and wherever the sort has put it.
#include "common.h"
#include "tile_fma.h"

// One wave a token: lane l holds the logits of experts l, l + 64, ...; `top` rounds of "the largest not taken yet"
// (the lowest index among equals), each a maximum over the wave.
#define RT_PER_LANE 16        // experts a lane holds: E <= 64 * RT_PER_LANE
__global__ __launch_bounds__(256) void router_topk_kernel(const float* __restrict__ logits,
                                                          const void* __restrict__ bias, int bias_dtype,
                                                          int* __restrict__ ids, float* __restrict__ weights, int N,
                                                          int E, int top) {
  const int n = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (n >= N) return;
  const float* z = logits + (size_t)n * E;
  float v[RT_PER_LANE];
  unsigned taken = 0u;
#pragma unroll
  for (int c = 0; c < RT_PER_LANE; ++c) {
    const int e = lane + 64 * c;
    v[c] = e < E ? z[e] + (bias ? load_as_float(bias, bias_dtype, e) : 0.f) : -INFINITY;
    if (e >= E) taken |= 1u << c;
  }
  float first_v = 0.f, sum = 0.f;
  for (int k = 0; k < top; ++k) {
    float best_v = -INFINITY;
    int best_e = 0x7fffffff;
#pragma unroll
    for (int c = 0; c < RT_PER_LANE; ++c) {
      const bool free_ = !((taken >> c) & 1u);
      // a value that compares with nothing (NaN) counts as the smallest
      const float x = (v[c] == v[c]) ? v[c] : -INFINITY;
      if (free_ && (best_e == 0x7fffffff || x > best_v)) { best_v = x; best_e = lane + 64 * c; }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(best_v, o, IA_WAVE);
      const int oe = __shfl_xor(best_e, o, IA_WAVE);
      if (oe != 0x7fffffff && (best_e == 0x7fffffff || ov > best_v || (ov == best_v && oe < best_e))) {
        best_v = ov;
        best_e = oe;
      }
    }
    if ((best_e & 63) == lane) taken |= 1u << (best_e >> 6);
    if (k == 0) first_v = best_v;
    const float w = expf(best_v - first_v);
    sum += w;
    if (lane == 0) {
      ids[(size_t)n * top + k] = best_e;
      weights[(size_t)n * top + k] = w;
    }
  }
  const float inv = 1.0f / sum;
  if (lane == 0)
    for (int k = 0; k < top; ++k) weights[(size_t)n * top + k] *= inv;
}

extern "C" int ia_router_topk(const float* logits, const void* bias, int bias_dtype, int* ids, float* weights, int N,
                              int E, int top, hipStream_t stream) {
  if (N < 0 || E <= 0 || top <= 0 || top > E) return IA_ERR_BAD_ARG;
  if (E > 64 * RT_PER_LANE) return IA_ERR_UNSUPPORTED;
  if (N == 0) return IA_OK;
  router_topk_kernel<<<(N + 3) / 4, 256, 0, stream>>>(logits, bias, bias_dtype, ids, weights, N, E, top);
  IA_LAUNCH_CHECK();
  return IA_OK;
}

#define MOE_MAX_E 1024
// One workgroup.  offsets[e] .. offsets[e + 1] - 1 are the places in perm of expert e's pairs; the order of an
// expert's pairs is whatever the atomics give (no result depends on it).
__global__ __launch_bounds__(1024) void moe_sort_kernel(const int* __restrict__ ids, int* __restrict__ offsets,
                                                        int* __restrict__ perm, int P, int E) {
  __shared__ int cnt[MOE_MAX_E];
  __shared__ int cur[MOE_MAX_E];
  for (int e = threadIdx.x; e < E; e += 1024) cnt[e] = 0;
  __syncthreads();
  for (int p = threadIdx.x; p < P; p += 1024) {
    const int e = ids[p];
    if ((unsigned)e < (unsigned)E) atomicAdd(&cnt[e], 1);
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    int at = 0;
    for (int e = 0; e < E; ++e) {
      offsets[e] = at;
      cur[e] = at;
      at += cnt[e];
    }
    offsets[E] = at;
  }
  __syncthreads();
  for (int p = threadIdx.x; p < P; p += 1024) {
    const int e = ids[p];
    if ((unsigned)e < (unsigned)E) perm[atomicAdd(&cur[e], 1)] = p;
  }
}

extern "C" int ia_moe_sort(const int* ids, int* offsets, int* perm, int P, int E, hipStream_t stream) {
  if (P < 0 || E <= 0) return IA_ERR_BAD_ARG;
  if (E > MOE_MAX_E) return IA_ERR_UNSUPPORTED;
  moe_sort_kernel<<<1, 1024, 0, stream>>>(ids, offsets, perm, P, E);
  IA_LAUNCH_CHECK();
  return IA_OK;
}

// Tile t of the launch (`rows` pairs a tile, expert by expert): its expert and its first place in perm; false when
// the launch has more tiles than the step needs.
__device__ __forceinline__ bool moe_tile(const int* __restrict__ offsets, int E, int t, int& expert, int& first,
                                         int& last, int rows = TF_T) {
  int seen = 0;
  for (int e = 0; e < E; ++e) {
    const int lo = offsets[e], hi = offsets[e + 1];
    const int tiles = (hi - lo + rows - 1) / rows;
    if (t < seen + tiles) {
      expert = e;
      first = lo + (t - seen) * rows;
      last = hi;
      return true;
    }
    seen += tiles;
  }
  return false;
}

// grid: (tiles of 2 * ff columns, ceil(P / 64) + E).  Wgu [E, 2 ff, W]: row 2 j the gate's row j, row 2 j + 1 up's.
// On the vector ALUs in fp32: the 32-bit path, and bfloat16 rows that cannot be read 16 bytes at a time.
template <typename T>
__global__ __launch_bounds__(256) void moe_gate_up_kernel(const T* __restrict__ x, const T* __restrict__ Wgu,
                                                          T* __restrict__ y, const int* __restrict__ offsets,
                                                          const int* __restrict__ perm, int E, int top, int W,
                                                          int ff, float limit, float alpha, float shift,
                                                          const float* __restrict__ in_w) {
  __shared__ TileFmaLds lds;
  int e, first, last;
  if (!moe_tile(offsets, E, blockIdx.y, e, first, last)) return;
  const int n0 = blockIdx.x * TF_T;
  const int lr = threadIdx.x >> 2;
  const T* a_row = (first + lr < last) ? x + (size_t)(perm[first + lr] / top) * W : nullptr;
  const T* w_row = (n0 + lr < 2 * ff) ? Wgu + ((size_t)e * 2 * ff + n0 + lr) * W : nullptr;
  tile_64(a_row, w_row, W, lds, [&](int i, int j0, const float* v) {
    const int p = first + i;
    if (p >= last) return;
    const float wt = in_w ? in_w[perm[p]] : 1.0f;
#pragma unroll
    for (int j = 0; j < 4; j += 2) {
      const int c = n0 + j0 + j;
      if (c + 1 >= 2 * ff) continue;
      // both products are rounded as a stored tensor would be, then the activation in fp32
      const float g = fminf(wt * to_float(from_float<T>(v[j])), limit);
      const float u = fminf(fmaxf(wt * to_float(from_float<T>(v[j + 1])), -limit), limit);
      y[(size_t)p * ff + (c >> 1)] = from_float<T>(g * (1.0f / (1.0f + expf(-alpha * g))) * (u + shift));
    }
  });
}

// The same on tiles of BM x BN (tile_mfma_big): grid (tiles of BN of the 2 ff columns, ceil(P / BM) + E).
template <int BM, int BN>
__global__ __launch_bounds__(BN == 256 ? 512 : 256) void moe_gate_up_big_kernel(const bf16_t* __restrict__ x, const bf16_t* __restrict__ Wgu,
                                                              bf16_t* __restrict__ y, const int* __restrict__ offsets,
                                                              const int* __restrict__ perm, int E, int top, int W,
                                                              int ff, float limit, float alpha, float shift,
                                                              const float* __restrict__ in_w) {
  __shared__ TileBigLds<BM, BN> lds;
  int e, first, last;
  if (!moe_tile(offsets, E, blockIdx.y, e, first, last, BM)) return;
  const int n0 = blockIdx.x * BN;
  tile_mfma_big<BM, BN>(
      [&](int r) { return x + (size_t)(perm[first + r] / top) * W; },
      [&](int r) { return Wgu + ((size_t)e * 2 * ff + n0 + r) * W; }, last - first, 2 * ff - n0, W, lds,
      [&](int i, int j0, const float* v) {
        const int p = first + i;
        if (p >= last) return;
        const float wt = in_w ? in_w[perm[p]] : 1.0f;
#pragma unroll
        for (int j = 0; j < 4; j += 2) {
          const int c = n0 + j0 + j;
          if (c + 1 >= 2 * ff) continue;
          const float g = fminf(wt * to_float(from_float<bf16_t>(v[j])), limit);
          const float u = fminf(fmaxf(wt * to_float(from_float<bf16_t>(v[j + 1])), -limit), limit);
          y[(size_t)p * ff + (c >> 1)] = from_float<bf16_t>(g * (1.0f / (1.0f + expf(-alpha * g))) * (u + shift));
        }
      });
}

// Rows a tile of the experts' products takes: 128 where an expert has some tens of pairs on average, else 32.
static inline int moe_tile_rows(int P, int E) { return (long)P >= 48L * E ? 128 : 32; }

extern "C" int ia_moe_gate_up(const void* x, const void* Wgu, void* y, const int* offsets, const int* perm, int dtype,
                              int P, int E, int top, int W, int ff, float limit, float alpha, float shift,
                              const float* in_weights, hipStream_t stream) {
  if (P < 0 || E <= 0 || top <= 0 || W <= 0 || ff <= 0) return IA_ERR_BAD_ARG;
  if (P == 0) return IA_OK;
  dim3 grid((2 * ff + TF_T - 1) / TF_T, (P + TF_T - 1) / TF_T + E);
  if (grid.y > 65535u) return IA_ERR_UNSUPPORTED;
  if (dtype == IA_F32)
    moe_gate_up_kernel<float><<<grid, 256, 0, stream>>>((const float*)x, (const float*)Wgu, (float*)y, offsets,
                                                               perm, E, top, W, ff, limit, alpha, shift, in_weights);
  else if (dtype == IA_BF16 && tile_rows_aligned(x, W) && tile_rows_aligned(Wgu, W)) {
    const int bm = moe_tile_rows(P, E);
    const int bn = bm == 128 ? 256 : TB_N;
    dim3 big((2 * ff + bn - 1) / bn, (P + bm - 1) / bm + E);
    if (big.y > 65535u) return IA_ERR_UNSUPPORTED;
    if (bm == 128)
      moe_gate_up_big_kernel<128, 256><<<big, 512, 0, stream>>>((const bf16_t*)x, (const bf16_t*)Wgu, (bf16_t*)y, offsets,
                                                           perm, E, top, W, ff, limit, alpha, shift, in_weights);
    else
      moe_gate_up_big_kernel<32, TB_N><<<big, 256, 0, stream>>>((const bf16_t*)x, (const bf16_t*)Wgu, (bf16_t*)y, offsets,
                                                          perm, E, top, W, ff, limit, alpha, shift, in_weights);
  }
  else if (dtype == IA_BF16)
    moe_gate_up_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)x, (const bf16_t*)Wgu, (bf16_t*)y,
                                                                offsets, perm, E, top, W, ff, limit, alpha, shift, in_weights);
  else
    return IA_ERR_BAD_ARG;
  IA_LAUNCH_CHECK();
  return IA_OK;
}

// grid: (tiles of W columns, ceil(P / 64) + E).  Wd [E, W, ff]; parts [top, N, W] fp32.
template <typename T>
__global__ __launch_bounds__(256) void moe_down_kernel(const T* __restrict__ y, const T* __restrict__ Wd,
                                                       float* __restrict__ parts, const float* __restrict__ weights,
                                                       const int* __restrict__ offsets, const int* __restrict__ perm,
                                                       int E, int top, int N, int W, int ff) {
  __shared__ TileFmaLds lds;
  int e, first, last;
  if (!moe_tile(offsets, E, blockIdx.y, e, first, last)) return;
  const int n0 = blockIdx.x * TF_T;
  const int lr = threadIdx.x >> 2;
  const T* a_row = (first + lr < last) ? y + (size_t)(first + lr) * ff : nullptr;
  const T* w_row = (n0 + lr < W) ? Wd + ((size_t)e * W + n0 + lr) * ff : nullptr;
  tile_64(a_row, w_row, ff, lds, [&](int i, int j0, const float* v) {
    const int p = first + i;
    if (p >= last) return;
    const int pair = perm[p];
    const int token = pair / top, choice = pair - token * top;
    const float wt = weights ? weights[pair] : 1.0f;
    float* o = parts + ((size_t)choice * N + token) * W;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = n0 + j0 + j;
      if (c < W) o[c] = to_float(from_float<T>(v[j])) * wt;
    }
  });
}

template <int BM, int BN>
__global__ __launch_bounds__(BN == 256 ? 512 : 256) void moe_down_big_kernel(const bf16_t* __restrict__ y, const bf16_t* __restrict__ Wd,
                                                           float* __restrict__ parts, const float* __restrict__ weights,
                                                           const int* __restrict__ offsets, const int* __restrict__ perm,
                                                           int E, int top, int N, int W, int ff) {
  __shared__ TileBigLds<BM, BN> lds;
  int e, first, last;
  if (!moe_tile(offsets, E, blockIdx.y, e, first, last, BM)) return;
  const int n0 = blockIdx.x * BN;
  tile_mfma_big<BM, BN>(
      [&](int r) { return y + (size_t)(first + r) * ff; },
      [&](int r) { return Wd + ((size_t)e * W + n0 + r) * ff; }, last - first, W - n0, ff, lds,
      [&](int i, int j0, const float* v) {
        const int p = first + i;
        if (p >= last) return;
        const int pair = perm[p];
        const int token = pair / top, choice = pair - token * top;
        const float wt = weights ? weights[pair] : 1.0f;
        float* o = parts + ((size_t)choice * N + token) * W;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int c = n0 + j0 + j;
          if (c < W) o[c] = to_float(from_float<bf16_t>(v[j])) * wt;
        }
      });
}

extern "C" int ia_moe_down(const void* y, const void* Wd, float* parts, const float* weights, const int* offsets,
                           const int* perm, int dtype, int N, int E, int top, int W, int ff, hipStream_t stream) {
  if (N < 0 || E <= 0 || top <= 0 || W <= 0 || ff <= 0) return IA_ERR_BAD_ARG;
  if (N == 0) return IA_OK;
  const int P = N * top;
  dim3 grid((W + TF_T - 1) / TF_T, (P + TF_T - 1) / TF_T + E);
  if (grid.y > 65535u) return IA_ERR_UNSUPPORTED;
  if (dtype == IA_F32)
    moe_down_kernel<float><<<grid, 256, 0, stream>>>((const float*)y, (const float*)Wd, parts, weights, offsets,
                                                            perm, E, top, N, W, ff);
  else if (dtype == IA_BF16 && tile_rows_aligned(y, ff) && tile_rows_aligned(Wd, ff)) {
    const int bm = moe_tile_rows(P, E);
    const int bn = bm == 128 ? 256 : TB_N;
    dim3 big((W + bn - 1) / bn, (P + bm - 1) / bm + E);
    if (big.y > 65535u) return IA_ERR_UNSUPPORTED;
    if (bm == 128)
      moe_down_big_kernel<128, 256><<<big, 512, 0, stream>>>((const bf16_t*)y, (const bf16_t*)Wd, parts, weights, offsets,
                                                        perm, E, top, N, W, ff);
    else
      moe_down_big_kernel<32, TB_N><<<big, 256, 0, stream>>>((const bf16_t*)y, (const bf16_t*)Wd, parts, weights, offsets,
                                                       perm, E, top, N, W, ff);
  }
  else if (dtype == IA_BF16)
    moe_down_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)y, (const bf16_t*)Wd, parts, weights,
                                                             offsets, perm, E, top, N, W, ff);
  else
    return IA_ERR_BAD_ARG;
  IA_LAUNCH_CHECK();
  return IA_OK;
}

// ---- the experts of a step of many rows by the grouped form of the LDS-tiled product (ia_gemm_mfma_grouped) ----------
// The tokens' rows are first brought into the order of the sort (an expert's rows one after the other), the two
// products run expert by expert over those rows, and the activation and the routing weight are passes of their own:
//   ia_moe_gather   xs[p, :] = x[perm[p] / top, :]
//   ia_moe_glu      y[p, j] = g sigmoid(alpha g) (u + shift), g = min(gu[p, 2 j], limit), u = clamp(gu[p, 2 j + 1], +-limit)
//   ia_moe_scatter  parts[choice, token, :] = float(o[p, :]) * weights[perm[p]], for the places p below *last (nullable:
//                   all of them)
// All three in bfloat16 with rows that are read 16 bytes at a time.
__global__ __launch_bounds__(256) void moe_gather_kernel(const uint4* __restrict__ x, const int* __restrict__ perm,
                                                         uint4* __restrict__ xs, int top, int pieces) {
  const int p = blockIdx.x;
  const uint4* src = x + (size_t)(perm[p] / top) * pieces;
  uint4* dst = xs + (size_t)p * pieces;
  for (int i = threadIdx.x; i < pieces; i += 256) dst[i] = src[i];
}

extern "C" int ia_moe_gather(const void* x, const int* perm, void* xs, int P, int top, int W, hipStream_t stream) {
  if (P < 0 || top <= 0 || W <= 0) return IA_ERR_BAD_ARG;
  if ((W & 7) || ((reinterpret_cast<uintptr_t>(x) | reinterpret_cast<uintptr_t>(xs)) & 15)) return IA_ERR_UNSUPPORTED;
  if (P == 0) return IA_OK;
  moe_gather_kernel<<<P, 256, 0, stream>>>((const uint4*)x, perm, (uint4*)xs, top, W / 8);
  IA_LAUNCH_CHECK();
  return IA_OK;
}

__global__ __launch_bounds__(256) void moe_glu_kernel(const uint4* __restrict__ gu, uint2* __restrict__ y, size_t n4,
                                                      float limit, float alpha, float shift, const int* __restrict__ perm,
                                                      const float* __restrict__ in_w, int quads) {
  const size_t stride = (size_t)gridDim.x * 256;
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n4; i += stride) {
    const uint4 v = gu[i];
    const uint32_t w[4] = {v.x, v.y, v.z, v.w};
    float o[4];
    const float wt = in_w ? in_w[perm[i / quads]] : 1.0f;
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const float g = fminf(wt * __uint_as_float(w[k] << 16), limit);
      const float u = fminf(fmaxf(wt * __uint_as_float(w[k] & 0xffff0000u), -limit), limit);
      o[k] = g * (1.0f / (1.0f + expf(-alpha * g))) * (u + shift);
    }
    uint2 r;
    r.x = (uint32_t)float_to_bf16_bits(o[0]) | ((uint32_t)float_to_bf16_bits(o[1]) << 16);
    r.y = (uint32_t)float_to_bf16_bits(o[2]) | ((uint32_t)float_to_bf16_bits(o[3]) << 16);
    y[i] = r;
  }
}

extern "C" int ia_moe_glu(const void* gu, void* y, int P, int ff, float limit, float alpha, float shift, const int* perm,
                          const float* in_weights, hipStream_t stream) {
  if (P < 0 || ff <= 0 || (in_weights && !perm)) return IA_ERR_BAD_ARG;
  if ((ff & 3) || ((reinterpret_cast<uintptr_t>(gu) | reinterpret_cast<uintptr_t>(y)) & 15)) return IA_ERR_UNSUPPORTED;
  const size_t n4 = (size_t)P * ff / 4;
  if (n4 == 0) return IA_OK;
  const unsigned grid = (unsigned)((n4 + 255) / 256 < 65536 ? (n4 + 255) / 256 : 65536);
  moe_glu_kernel<<<grid, 256, 0, stream>>>((const uint4*)gu, (uint2*)y, n4, limit, alpha, shift, perm, in_weights, ff / 4);
  IA_LAUNCH_CHECK();
  return IA_OK;
}

__global__ __launch_bounds__(256) void moe_scatter_kernel(const uint4* __restrict__ o, const int* __restrict__ perm,
                                                          const float* __restrict__ weights, float* __restrict__ parts,
                                                          const int* __restrict__ last, int N, int top, int W) {
  const int p = blockIdx.x;
  if (last && p >= *last) return;                  // a pair that went to no expert with tensors
  const int pair = perm[p];
  const int token = pair / top, choice = pair - token * top;
  const float wt = weights ? weights[pair] : 1.0f;
  const uint4* src = o + (size_t)p * (W / 8);
  float4* dst = reinterpret_cast<float4*>(parts + ((size_t)choice * N + token) * W);
  for (int i = threadIdx.x; i < W / 8; i += 256) {
    const uint4 v = src[i];
    dst[2 * i] = make_float4(__uint_as_float(v.x << 16) * wt, __uint_as_float(v.x & 0xffff0000u) * wt,
                             __uint_as_float(v.y << 16) * wt, __uint_as_float(v.y & 0xffff0000u) * wt);
    dst[2 * i + 1] = make_float4(__uint_as_float(v.z << 16) * wt, __uint_as_float(v.z & 0xffff0000u) * wt,
                                 __uint_as_float(v.w << 16) * wt, __uint_as_float(v.w & 0xffff0000u) * wt);
  }
}

extern "C" int ia_moe_scatter(const void* o, const int* perm, const float* weights, float* parts, const int* last, int N,
                              int top, int W, hipStream_t stream) {
  if (N < 0 || top <= 0 || W <= 0) return IA_ERR_BAD_ARG;
  if ((W & 7) || ((reinterpret_cast<uintptr_t>(o) | reinterpret_cast<uintptr_t>(parts)) & 15)) return IA_ERR_UNSUPPORTED;
  if (N == 0) return IA_OK;
  moe_scatter_kernel<<<N * top, 256, 0, stream>>>((const uint4*)o, perm, weights, parts, last, N, top, W);
  IA_LAUNCH_CHECK();
  return IA_OK;
}

// ---- experts without a gate, and a router whose choice and weights go by different numbers ----
//   ia_router_softmax_topk   s = softmax(z) over all experts; the `top` largest of s + correction are chosen (the
//                            lowest index among equals); the weights are the chosen s, with `renorm` over their sum
//                            (+ 1e-20).  With `sigmoid` s = sigmoid(z) instead, and without a correction the choice goes
//                            by z itself (large z have equal s in fp32).  With `groups` > 1 the experts form that many groups of neighbours, a group's
//                            score is its largest s + correction, and only experts of the `keep` best groups (the
//                            lowest index among equals) can be chosen;
//   ia_moe_up                per expert, over its pairs' tokens: y = act(Wu x), Wu [E, ff, W]; act by the codes of
//                            ia_activation (2: the erf GELU, 3: the square of relu).
__device__ __forceinline__ float moe_act(float z, int act) {
  if (act == 3) { const float r = fmaxf(z, 0.f); return r * r; }
  if (act == 2) return 0.5f * z * (1.0f + erff(z * 0.7071067811865476f));
  if (act == 1) return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
  return z;
}

// PL: experts a lane holds (lane, lane + 64, ...)
template <int PL>
__global__ __launch_bounds__(256) void router_softmax_topk_kernel(const float* __restrict__ logits,
                                                                  const void* __restrict__ corr, int corr_dtype,
                                                                  int* __restrict__ ids, float* __restrict__ weights,
                                                                  int N, int E, int top, int z_stride, int groups,
                                                                  int keep, int renorm, int sigmoid) {
  __shared__ float s_v[4][64 * PL];       // a wave's choice scores, then (in place) its groups' scores
  const int n = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (n >= N) return;
  const float* z = logits + (size_t)n * z_stride;
  float s[PL], v[PL];
  unsigned taken = 0u;
  float zmax = -INFINITY;
#pragma unroll
  for (int c = 0; c < PL; ++c) {
    const int e = lane + 64 * c;
    s[c] = e < E ? z[e] : -INFINITY;
    zmax = fmaxf(zmax, s[c]);
    if (e >= E) taken |= 1u << c;
  }
  zmax = wave_max(zmax);
  float total = 0.f;
#pragma unroll
  for (int c = 0; c < PL; ++c) {
    s[c] = (lane + 64 * c) < E ? expf(s[c] - zmax) : 0.f;
    total += s[c];
  }
  total = wave_sum(total);
  const float inv_total = 1.0f / total;
#pragma unroll
  for (int c = 0; c < PL; ++c) {
    const int e = lane + 64 * c;
    if (sigmoid) {
      const float x = e < E ? z[e] : -INFINITY;
      s[c] = 1.0f / (1.0f + expf(-x));
      v[c] = e < E ? (corr ? s[c] + load_as_float(corr, corr_dtype, e) : x) : -INFINITY;
    } else {
      s[c] *= inv_total;
      v[c] = e < E ? s[c] + (corr ? load_as_float(corr, corr_dtype, e) : 0.f) : -INFINITY;
    }
  }
  if (groups > 1) {
    // each wave works on its own part of LDS: a wave's accesses are in order, no barrier is needed between them
    volatile float* mine = s_v[threadIdx.x >> 6];
    const int size = E / groups;
#pragma unroll
    for (int c = 0; c < PL; ++c)
      if (lane + 64 * c < E) mine[lane + 64 * c] = (v[c] == v[c]) ? v[c] : -INFINITY;
    float gs[PL];                        // this lane's groups: lane, lane + 64, ...
#pragma unroll
    for (int c = 0; c < PL; ++c) {
      gs[c] = -INFINITY;
      const int g = lane + 64 * c;
      if (g < groups)
        for (int i = 0; i < size; ++i) gs[c] = fmaxf(gs[c], mine[g * size + i]);
    }
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int c = 0; c < PL; ++c)
      if (lane + 64 * c < groups) mine[lane + 64 * c] = gs[c];
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int c = 0; c < PL; ++c) {
      const int e = lane + 64 * c;
      if (e >= E) continue;
      const int g = e / size;
      const float own = mine[g];
      int better = 0;
      for (int i = 0; i < groups; ++i) better += mine[i] > own || (mine[i] == own && i < g);
      if (better >= keep) taken |= 1u << c;
    }
  }
  float sum = 0.f;
  for (int k = 0; k < top; ++k) {
    float best_v = -INFINITY, best_s = 0.f;
    int best_e = 0x7fffffff;
#pragma unroll
    for (int c = 0; c < PL; ++c) {
      const bool free_ = !((taken >> c) & 1u);
      const float x = (v[c] == v[c]) ? v[c] : -INFINITY;
      if (free_ && (best_e == 0x7fffffff || x > best_v)) { best_v = x; best_e = lane + 64 * c; best_s = s[c]; }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(best_v, o, IA_WAVE), os = __shfl_xor(best_s, o, IA_WAVE);
      const int oe = __shfl_xor(best_e, o, IA_WAVE);
      if (oe != 0x7fffffff && (best_e == 0x7fffffff || ov > best_v || (ov == best_v && oe < best_e))) {
        best_v = ov;
        best_e = oe;
        best_s = os;
      }
    }
    if ((best_e & 63) == lane) taken |= 1u << (best_e >> 6);
    sum += best_s;
    if (lane == 0) {
      ids[(size_t)n * top + k] = best_e;
      weights[(size_t)n * top + k] = best_s;
    }
  }
  const float inv = 1.0f / (sum + 1e-20f);
  if (lane == 0 && renorm)
    for (int k = 0; k < top; ++k) weights[(size_t)n * top + k] *= inv;
}

extern "C" int ia_router_softmax_topk(const float* logits, const void* corr, int corr_dtype, int* ids, float* weights,
                                      int N, int E, int top, int z_stride, int groups, int keep, int renorm,
                                      int sigmoid, hipStream_t stream) {
  if (N < 0 || E <= 0 || top <= 0 || top > E || z_stride < E || groups < 1 || E % groups || keep < 1 || keep > groups ||
      top > keep * (E / groups) || !logits || !ids || !weights) return IA_ERR_BAD_ARG;
  if (E > 64 * RT_PER_LANE) return IA_ERR_UNSUPPORTED;
  if (N == 0) return IA_OK;
#define IA_RT(PL)                                                                                                        \
  router_softmax_topk_kernel<PL><<<(N + 3) / 4, 256, 0, stream>>>(logits, corr, corr_dtype, ids, weights, N, E, top, z_stride, \
                                                                  groups, keep, renorm, sigmoid)
  if (E <= 64) IA_RT(1);
  else if (E <= 256) IA_RT(4);
  else IA_RT(RT_PER_LANE);
#undef IA_RT
  IA_LAUNCH_CHECK();
  return IA_OK;
}

template <typename T>
__global__ __launch_bounds__(256) void moe_up_kernel(const T* __restrict__ x, const T* __restrict__ Wu, T* __restrict__ y,
                                                     const int* __restrict__ offsets, const int* __restrict__ perm,
                                                     int E, int top, int W, int ff, int act) {
  __shared__ TileFmaLds lds;
  int e, first, last;
  if (!moe_tile(offsets, E, blockIdx.y, e, first, last)) return;
  const int n0 = blockIdx.x * TF_T;
  const int lr = threadIdx.x >> 2;
  const T* a_row = (first + lr < last) ? x + (size_t)(perm[first + lr] / top) * W : nullptr;
  const T* w_row = (n0 + lr < ff) ? Wu + ((size_t)e * ff + n0 + lr) * W : nullptr;
  tile_64(a_row, w_row, W, lds, [&](int i, int j0, const float* v) {
    const int p = first + i;
    if (p >= last) return;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = n0 + j0 + j;
      // the product is rounded as a stored tensor would be, then the activation in fp32
      if (c < ff) y[(size_t)p * ff + c] = from_float<T>(moe_act(to_float(from_float<T>(v[j])), act));
    }
  });
}

template <int BM, int BN>
__global__ __launch_bounds__(BN == 256 ? 512 : 256) void moe_up_big_kernel(const bf16_t* __restrict__ x, const bf16_t* __restrict__ Wu,
                                                              bf16_t* __restrict__ y, const int* __restrict__ offsets,
                                                              const int* __restrict__ perm, int E, int top, int W,
                                                              int ff, int act) {
  __shared__ TileBigLds<BM, BN> lds;
  int e, first, last;
  if (!moe_tile(offsets, E, blockIdx.y, e, first, last, BM)) return;
  const int n0 = blockIdx.x * BN;
  tile_mfma_big<BM, BN>(
      [&](int r) { return x + (size_t)(perm[first + r] / top) * W; },
      [&](int r) { return Wu + ((size_t)e * ff + n0 + r) * W; }, last - first, ff - n0, W, lds,
      [&](int i, int j0, const float* v) {
        const int p = first + i;
        if (p >= last) return;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int c = n0 + j0 + j;
          if (c < ff) y[(size_t)p * ff + c] = from_float<bf16_t>(moe_act(to_float(from_float<bf16_t>(v[j])), act));
        }
      });
}

extern "C" int ia_moe_up(const void* x, const void* Wu, void* y, const int* offsets, const int* perm, int dtype, int P,
                         int E, int top, int W, int ff, int act, hipStream_t stream) {
  if (P < 0 || E <= 0 || top <= 0 || W <= 0 || ff <= 0 || act < 0 || act > 3) return IA_ERR_BAD_ARG;
  if (P == 0) return IA_OK;
  dim3 grid((ff + TF_T - 1) / TF_T, (P + TF_T - 1) / TF_T + E);
  if (grid.y > 65535u) return IA_ERR_UNSUPPORTED;
  if (dtype == IA_F32)
    moe_up_kernel<float><<<grid, 256, 0, stream>>>((const float*)x, (const float*)Wu, (float*)y, offsets, perm, E, top,
                                                   W, ff, act);
  else if (dtype == IA_BF16 && tile_rows_aligned(x, W) && tile_rows_aligned(Wu, W)) {
    const int bm = moe_tile_rows(P, E);
    const int bn = bm == 128 ? 256 : TB_N;
    dim3 big((ff + bn - 1) / bn, (P + bm - 1) / bm + E);
    if (big.y > 65535u) return IA_ERR_UNSUPPORTED;
    if (bm == 128)
      moe_up_big_kernel<128, 256><<<big, 512, 0, stream>>>((const bf16_t*)x, (const bf16_t*)Wu, (bf16_t*)y, offsets, perm,
                                                           E, top, W, ff, act);
    else
      moe_up_big_kernel<32, TB_N><<<big, 256, 0, stream>>>((const bf16_t*)x, (const bf16_t*)Wu, (bf16_t*)y, offsets, perm,
                                                          E, top, W, ff, act);
  } else if (dtype == IA_BF16)
    moe_up_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)x, (const bf16_t*)Wu, (bf16_t*)y, offsets, perm, E,
                                                    top, W, ff, act);
  else
    return IA_ERR_BAD_ARG;
  IA_LAUNCH_CHECK();
  return IA_OK;
}

// ---- what a step adds beside its experts' products ----
//   ia_moe_extras   for every pair whose expert is one of the last, without tensors (ids >= E: an expert whose result is
//                   its input): parts[choice, token, :] = weight * x[token, :]; and for every token, with `shared`: its
//                   result ([splits, shared_rows, W], added in the order of the parts) times sigmoid(gate[token]) into
//                   parts[top, token, :], the part after the choices'.
// grid (N, top (+ 1), pieces of 256 V values of a row); V 4: rows of a multiple of four values, 16 (or 8) bytes an access.
__device__ __forceinline__ void mx_load(const float* p, float (&v)[1]) { v[0] = p[0]; }
__device__ __forceinline__ void mx_load(const bf16_t* p, float (&v)[1]) { v[0] = to_float(p[0]); }
__device__ __forceinline__ void mx_load(const float* p, float (&v)[4]) {
  const float4 t = *reinterpret_cast<const float4*>(p);
  v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
}
__device__ __forceinline__ void mx_load(const bf16_t* p, float (&v)[4]) {
  const uint2 t = *reinterpret_cast<const uint2*>(p);
  v[0] = __uint_as_float(t.x << 16); v[1] = __uint_as_float(t.x & 0xffff0000u);
  v[2] = __uint_as_float(t.y << 16); v[3] = __uint_as_float(t.y & 0xffff0000u);
}
__device__ __forceinline__ void mx_store(float* p, const float (&v)[1], float f) { p[0] = f * v[0]; }
__device__ __forceinline__ void mx_store(float* p, const float (&v)[4], float f) {
  *reinterpret_cast<float4*>(p) = make_float4(f * v[0], f * v[1], f * v[2], f * v[3]);
}

template <typename T, typename TS, int V>
__global__ __launch_bounds__(256) void moe_extras_kernel(const T* __restrict__ x, const int* __restrict__ ids,
                                                         const float* __restrict__ weights, float* __restrict__ parts,
                                                         const TS* __restrict__ shared, int splits, size_t split_stride,
                                                         const float* __restrict__ gate, int gate_stride, int N, int E,
                                                         int top, int W) {
  const int n = blockIdx.x, choice = blockIdx.y, i = (blockIdx.z * 256 + threadIdx.x) * V;
  float* o = parts + ((size_t)choice * N + n) * W + i;
  float v[V];
  if (choice == top) {
    if (i >= W) return;
    const TS* s = shared + (size_t)n * W + i;
    mx_load(s, v);
#pragma unroll 4
    for (int k = 1; k < splits; ++k) {                 // the parts in the order of their index
      float p[V];
      mx_load(s + k * split_stride, p);
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] += p[e];
    }
    mx_store(o, v, gate ? 1.0f / (1.0f + expf(-gate[(size_t)n * gate_stride])) : 1.0f);
    return;
  }
  if (ids[(size_t)n * top + choice] < E || i >= W) return;
  mx_load(x + (size_t)n * W + i, v);
  mx_store(o, v, weights[(size_t)n * top + choice]);
}

// parts: fp32 [top (+ 1 with shared), N, W]; shared (nullable) of shared_dtype; gate (nullable): fp32, token n's logit
// at gate[n gate_stride].
extern "C" int ia_moe_extras(const void* x, int dtype, const int* ids, const float* weights, float* parts, const void* shared,
                             int shared_dtype, int splits, int shared_rows, const float* gate, int gate_stride, int N, int E,
                             int top, int W, hipStream_t stream) {
  if (N < 0 || E < 0 || top <= 0 || W <= 0 || !x || !ids || !weights || !parts || top > 65534 ||
      (shared && (splits < 1 || shared_rows < N)) || (dtype != IA_F32 && dtype != IA_BF16) ||
      (shared && shared_dtype != IA_F32 && shared_dtype != IA_BF16))
    return IA_ERR_BAD_ARG;
  if (N == 0) return IA_OK;
  const bool vec = (W & 3) == 0 && (((uintptr_t)x | (uintptr_t)parts | (uintptr_t)shared) & 15) == 0;
  const dim3 grid(N, top + (shared ? 1 : 0), (W + (vec ? 1024 : 256) - 1) / (vec ? 1024 : 256));
  const size_t stride = (size_t)shared_rows * W;
#define IA_MX_V(T, TS, V)                                                                                                    \
  moe_extras_kernel<T, TS, V><<<grid, 256, 0, stream>>>((const T*)x, ids, weights, parts, (const TS*)shared, splits, stride, \
                                                        gate, gate_stride, N, E, top, W)
#define IA_MX(T, TS)                \
  do {                              \
    if (vec) IA_MX_V(T, TS, 4);     \
    else IA_MX_V(T, TS, 1);         \
  } while (0)
  const bool sf = !shared || shared_dtype == IA_F32;
  if (dtype == IA_F32) {
    if (sf) IA_MX(float, float);
    else return IA_ERR_BAD_ARG;
  } else if (sf) IA_MX(bf16_t, float);
  else IA_MX(bf16_t, bf16_t);
#undef IA_MX
#undef IA_MX_V
  IA_LAUNCH_CHECK();
  return IA_OK;
}

#include "op_call.h"
IA_OP(ia_moe_extras)
IA_OP(ia_router_topk)
IA_OP(ia_moe_sort)
IA_OP(ia_moe_gate_up)
IA_OP(ia_moe_down)
IA_OP(ia_moe_gather)
IA_OP(ia_moe_glu)
IA_OP(ia_moe_scatter)
IA_OP(ia_router_softmax_topk)
IA_OP(ia_moe_up)
