// Hyper-connections: S copies X_1 .. X_S of the residual stream side by side, [N, S, H] fp32.  A sublayer f reads a
// weighted sum of them, and its result goes back to all of them while they are mixed,
//     u = sum_s in[s] X_s,   y = f(g u / sqrt(mean(u^2) + eps)),   X_t <- sum_s mix[s][t] X_s + out[t] y,
// with the vectors in, out [S] and the matrix mix [from][to] of the sublayer (out already times whatever factor the
// model puts on its sublayers' results).
//
//   ia_hyper_step   one pass over the streams between two sublayers: writes back what the sublayer before left (y as a
//                   tensor, or as partial sums of a split product or of routed experts, added in the order of their
//                   index), forms the next sublayer's u from the new streams and leaves it normed and rounded once.
//                   Before the first sublayer the streams are all equal and need not exist: they are read from the one
//                   stream they are copies of.  After the last one their sum is left in place of a u.
//
// All of it fp32; a row's sums are taken in one order whatever the batch holds.
#include "common.h"

#define HY_MAX_S 32      // more than HY_FAST_S streams: a kernel whose loops over streams are not unrolled
#define HY_FAST_S 8
#define HY_KEEP 16       // values of a row that a thread of the plain kernel keeps in registers

struct HyperArgs {
  const float* src;      // streams [N, S, H], or with src_stream 0 one stream [N, H] that all are copies of
  size_t src_row, src_stream;
  float* streams;        // where the new streams go ([N, S, H]; may be src); not written without delta
  const void* delta;     // [splits, delta_rows, H] or null: nothing to write back
  size_t split_stride;
  const float* mix;      // [S, S], with delta
  const float* outw;     // [S], with delta
  const float* inw;      // [S] of the next sublayer; null: the plain sum
  const void* w;         // the norm's weight [H]; null: u itself goes to sum_out, fp32
  float* sum_out;        // [N, H]
  void* x;               // [N, H] in the activations' type
  int splits, w_dtype, H;
  float eps;
};

template <int S>
struct HyperWeights {
  float mix[S][S], outw[S], inw[S];
};

// The weights are the same for every row: read once through scalar loads into registers.
template <int S>
__device__ __forceinline__ void hyper_weights(const HyperArgs& A, HyperWeights<S>& W) {
#pragma unroll
  for (int t = 0; t < S; ++t) {
    W.outw[t] = A.delta ? A.outw[t] : 0.f;
    W.inw[t] = A.inw ? A.inw[t] : 1.f;
#pragma unroll
    for (int s = 0; s < S; ++s) W.mix[s][t] = A.delta ? A.mix[s * S + t] : (s == t ? 1.f : 0.f);
  }
}

// One value of every stream: the new values from the old ones and y, and u.
template <int S>
__device__ __forceinline__ float hyper_value(const HyperWeights<S>& W, const float (&x)[S], float y, bool has_delta,
                                             float (&n)[S]) {
  float u = 0.f;
#pragma unroll
  for (int t = 0; t < S; ++t) {
    if (has_delta) {
      float v = W.mix[0][t] * x[0];
#pragma unroll
      for (int s = 1; s < S; ++s) v = __builtin_fmaf(W.mix[s][t], x[s], v);
      n[t] = __builtin_fmaf(W.outw[t], y, v);
    } else {
      n[t] = x[t];
    }
    u = __builtin_fmaf(W.inw[t], n[t], u);
  }
  return u;
}

__device__ __forceinline__ float4 hy_load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 hy_load4(const bf16_t* p) {
  const uint2 u = *reinterpret_cast<const uint2*>(p);
  return make_float4(__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16),
                     __uint_as_float(u.y & 0xffff0000u));
}
__device__ __forceinline__ void hy_store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void hy_store4(bf16_t* p, float4 v) {
  uint2 u;
  u.x = (uint32_t)float_to_bf16_bits(v.x) | ((uint32_t)float_to_bf16_bits(v.y) << 16);
  u.y = (uint32_t)float_to_bf16_bits(v.z) | ((uint32_t)float_to_bf16_bits(v.w) << 16);
  *reinterpret_cast<uint2*>(p) = u;
}

// Rows of a multiple of 4 values up to NT * 4 * NV, 16 bytes a read; a workgroup a row, one pass over memory.
template <int S, typename TD, typename TX, int NT, int NV>
__global__ __launch_bounds__(NT) void hyper_vec_kernel(HyperArgs A) {
  __shared__ float red[NT / 64];
  const int row = blockIdx.x, H = A.H;
  const float* src = A.src + (size_t)row * A.src_row;
  float* dst = A.streams + (size_t)row * S * H;
  const TD* dr = reinterpret_cast<const TD*>(A.delta) + (size_t)row * H;
  const bool has_delta = A.delta != nullptr;
  HyperWeights<S> W;
  hyper_weights<S>(A, W);
  float4 u[NV];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < NV; ++c) {
    const int i = (threadIdx.x + c * NT) * 4;
    u[c] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (i < H) {
      float4 x[S], y = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
      for (int s = 0; s < S; ++s) x[s] = hy_load4(src + s * A.src_stream + i);
      if (has_delta) {
        y = hy_load4(dr + i);
#pragma unroll 4
        for (int k = 1; k < A.splits; ++k) {                  // the parts in the order of their index
          const float4 p = hy_load4(dr + k * A.split_stride + i);
          y.x += p.x; y.y += p.y; y.z += p.z; y.w += p.w;
        }
      }
      float n[4][S];
      const float yv[4] = {y.x, y.y, y.z, y.w};
      float uv[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        float xe[S];
#pragma unroll
        for (int s = 0; s < S; ++s) xe[s] = e == 0 ? x[s].x : (e == 1 ? x[s].y : (e == 2 ? x[s].z : x[s].w));
        uv[e] = hyper_value<S>(W, xe, yv[e], has_delta, n[e]);
      }
      if (has_delta && !A.sum_out) {
#pragma unroll
        for (int t = 0; t < S; ++t) hy_store4(dst + (size_t)t * H + i, make_float4(n[0][t], n[1][t], n[2][t], n[3][t]));
      }
      u[c] = make_float4(uv[0], uv[1], uv[2], uv[3]);
      ss += __builtin_fmaf(uv[0], uv[0], uv[1] * uv[1]) + __builtin_fmaf(uv[2], uv[2], uv[3] * uv[3]);
    }
  }
  if (A.sum_out) {
#pragma unroll
    for (int c = 0; c < NV; ++c) {
      const int i = (threadIdx.x + c * NT) * 4;
      if (i < H) hy_store4(A.sum_out + (size_t)row * H + i, u[c]);
    }
    return;
  }
  ss = block_sum<NT>(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)H + A.eps);
#pragma unroll
  for (int c = 0; c < NV; ++c) {
    const int i = (threadIdx.x + c * NT) * 4;
    if (i < H) {
      const float4 g = A.w_dtype == IA_F32 ? hy_load4((const float*)A.w + i) : hy_load4((const bf16_t*)A.w + i);
      hy_store4((TX*)A.x + (size_t)row * H + i,
                make_float4(u[c].x * inv * g.x, u[c].y * inv * g.y, u[c].z * inv * g.z, u[c].w * inv * g.w));
    }
  }
}

// Any row: values one at a time, those beyond 256 * HY_KEEP formed again from the streams just written.
template <int S, typename TD, typename TX>
__global__ __launch_bounds__(256) void hyper_kernel(HyperArgs A) {
  __shared__ float red[4];
  const int row = blockIdx.x, H = A.H;
  const float* src = A.src + (size_t)row * A.src_row;
  float* dst = A.streams + (size_t)row * S * H;
  const TD* dr = reinterpret_cast<const TD*>(A.delta) + (size_t)row * H;
  const bool has_delta = A.delta != nullptr;
  HyperWeights<S> W;
  hyper_weights<S>(A, W);
  auto value = [&](int i) {
    float x[S], n[S];
#pragma unroll
    for (int s = 0; s < S; ++s) x[s] = src[s * A.src_stream + i];
    const float y = has_delta ? load_split_sum(dr + i, A.splits, A.split_stride) : 0.f;
    const float u = hyper_value<S>(W, x, y, has_delta, n);
    if (has_delta && !A.sum_out) {
#pragma unroll
      for (int t = 0; t < S; ++t) dst[(size_t)t * H + i] = n[t];
    }
    return u;
  };
  if (A.sum_out) {
    for (int i = threadIdx.x; i < H; i += 256) A.sum_out[(size_t)row * H + i] = value(i);
    return;
  }
  float keep[HY_KEEP];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < HY_KEEP; ++c) {
    const int i = threadIdx.x + c * 256;
    keep[c] = i < H ? value(i) : 0.f;
    ss = __builtin_fmaf(keep[c], keep[c], ss);
  }
  for (int i = threadIdx.x + HY_KEEP * 256; i < H; i += 256) {
    const float u = value(i);
    ss = __builtin_fmaf(u, u, ss);
  }
  ss = block_sum<256>(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)H + A.eps);
  TX* x = (TX*)A.x + (size_t)row * H;
#pragma unroll
  for (int c = 0; c < HY_KEEP; ++c) {
    const int i = threadIdx.x + c * 256;
    if (i < H) x[i] = from_float<TX>(keep[c] * inv * load_as_float(A.w, A.w_dtype, i));
  }
  for (int i = threadIdx.x + HY_KEEP * 256; i < H; i += 256) {
    float u = 0.f;
#pragma unroll
    for (int t = 0; t < S; ++t)
      u = __builtin_fmaf(W.inw[t], has_delta ? dst[(size_t)t * H + i] : src[t * A.src_stream + i], u);
    x[i] = from_float<TX>(u * inv * load_as_float(A.w, A.w_dtype, i));
  }
}

// More streams than the kernels above are made for: a value at a time, the numbers of a value's streams in scratch.
template <typename TD, typename TX>
__global__ __launch_bounds__(256) void hyper_many_kernel(HyperArgs A, int S) {
  __shared__ float red[4];
  const int row = blockIdx.x, H = A.H;
  const float* src = A.src + (size_t)row * A.src_row;
  float* dst = A.streams + (size_t)row * S * H;
  const TD* dr = reinterpret_cast<const TD*>(A.delta) + (size_t)row * H;
  const bool has_delta = A.delta != nullptr;
  float ss = 0.f;
  for (int i = threadIdx.x; i < H; i += 256) {
    float x[HY_MAX_S];
    for (int s = 0; s < S; ++s) x[s] = src[s * A.src_stream + i];
    const float y = has_delta ? load_split_sum(dr + i, A.splits, A.split_stride) : 0.f;
    float u = 0.f;
    for (int t = 0; t < S; ++t) {
      float n = x[t];
      if (has_delta) {
        n = A.mix[t] * x[0];
        for (int s = 1; s < S; ++s) n = __builtin_fmaf(A.mix[s * S + t], x[s], n);
        n = __builtin_fmaf(A.outw[t], y, n);
        if (!A.sum_out) dst[(size_t)t * H + i] = n;
      }
      u = __builtin_fmaf(A.inw ? A.inw[t] : 1.f, n, u);
    }
    if (A.sum_out) A.sum_out[(size_t)row * H + i] = u;
    ss = __builtin_fmaf(u, u, ss);
  }
  if (A.sum_out) return;
  ss = block_sum<256>(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)H + A.eps);
  for (int i = threadIdx.x; i < H; i += 256) {              // u once more, from the streams this thread left
    float u = 0.f;
    for (int t = 0; t < S; ++t)
      u = __builtin_fmaf(A.inw ? A.inw[t] : 1.f, has_delta ? dst[(size_t)t * H + i] : src[t * A.src_stream + i], u);
    ((TX*)A.x)[(size_t)row * H + i] = from_float<TX>(u * inv * load_as_float(A.w, A.w_dtype, i));
  }
}

template <int S, typename TD, typename TX>
static int hyper_launch(const HyperArgs& A, int N, hipStream_t stream) {
  const bool aligned = ((reinterpret_cast<uintptr_t>(A.src) | reinterpret_cast<uintptr_t>(A.streams) |
                         reinterpret_cast<uintptr_t>(A.delta) | reinterpret_cast<uintptr_t>(A.w) |
                         reinterpret_cast<uintptr_t>(A.x) | reinterpret_cast<uintptr_t>(A.sum_out)) & 15) == 0;
  const int H = A.H;
  // the kernel follows from H alone: a row's sums are taken in one order
  if (aligned && (H & 3) == 0 && H <= 256 * 4) hyper_vec_kernel<S, TD, TX, 256, 1><<<N, 256, 0, stream>>>(A);
  else if (aligned && (H & 3) == 0 && H <= 512 * 4) hyper_vec_kernel<S, TD, TX, 512, 1><<<N, 512, 0, stream>>>(A);
  else if (aligned && (H & 3) == 0 && H <= 512 * 4 * 4) hyper_vec_kernel<S, TD, TX, 512, 4><<<N, 512, 0, stream>>>(A);
  else hyper_kernel<S, TD, TX><<<N, 256, 0, stream>>>(A);
  IA_LAUNCH_CHECK();
  return IA_OK;
}

template <int S>
static int hyper_types(const HyperArgs& A, int delta_dtype, int act_dtype, int N, hipStream_t stream) {
  if (act_dtype == IA_F32) return hyper_launch<S, float, float>(A, N, stream);
  if (delta_dtype == IA_F32) return hyper_launch<S, float, bf16_t>(A, N, stream);
  return hyper_launch<S, bf16_t, bf16_t>(A, N, stream);
}

// src_streams 0: src is ONE stream [N, H] that all S are copies of; otherwise [N, S, H].  delta (nullable): [splits,
// delta_rows, H] of delta_dtype, then mix, outw and (without sum_out) streams.  With w: x gets the normed u; without:
// sum_out gets u unrounded (inw null: the plain sum of the streams) and the streams are left as they were.
extern "C" int ia_hyper_step(const float* src, int src_streams, float* streams, const void* delta, int delta_dtype, int splits,
                             int delta_rows, const float* mix, const float* outw, const float* inw, const void* w,
                             int w_dtype, float* sum_out, void* x, int act_dtype, int N, int S, int H, float eps,
                             hipStream_t stream) {
  if (N < 0 || H <= 0 || S <= 0 || !src || (delta && (!mix || !outw || splits < 1 || delta_rows < N)) ||
      (w ? (!x || sum_out || !(eps > 0.f) || (delta && !streams)) : !sum_out) || (src_streams != 0 && src_streams != S) ||
      (act_dtype != IA_F32 && act_dtype != IA_BF16) ||
      (delta && !(delta_dtype == IA_F32 || (delta_dtype == IA_BF16 && act_dtype == IA_BF16))))
    return IA_ERR_BAD_ARG;
  if (S > HY_MAX_S) return IA_ERR_UNSUPPORTED;
  if (N == 0) return IA_OK;
  HyperArgs A;
  A.src = src;
  A.src_row = (size_t)(src_streams ? S : 1) * H;
  A.src_stream = src_streams ? (size_t)H : 0;
  A.streams = streams;
  A.delta = delta;
  A.split_stride = (size_t)delta_rows * H;
  A.mix = mix;
  A.outw = outw;
  A.inw = inw;
  A.w = w;
  A.sum_out = sum_out;
  A.x = x;
  A.splits = splits;
  A.w_dtype = w_dtype;
  A.H = H;
  A.eps = eps;
  switch (S) {
#define IA_HY(n) case n: return hyper_types<n>(A, delta_dtype, act_dtype, N, stream)
    IA_HY(1); IA_HY(2); IA_HY(3); IA_HY(4); IA_HY(5); IA_HY(6); IA_HY(7); IA_HY(8);
#undef IA_HY
  }
  if (act_dtype == IA_F32) hyper_many_kernel<float, float><<<N, 256, 0, stream>>>(A, S);
  else if (delta_dtype == IA_F32) hyper_many_kernel<float, bf16_t><<<N, 256, 0, stream>>>(A, S);
  else hyper_many_kernel<bf16_t, bf16_t><<<N, 256, 0, stream>>>(A, S);
  IA_LAUNCH_CHECK();
  return IA_OK;
}

#include "op_call.h"
IA_OP(ia_hyper_step)
