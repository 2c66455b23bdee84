// The selective scan with a decay per channel and state value (the Mamba-1 form):
//
//     dt = softplus(raw + bias_c),      S[n] <- exp(dt A[c, n]) S[n] + dt x_c B[n],      y_c = sum_n S[n] C[n] + D_c x_c,
//
// B and C shared by all channels of a token, the state fp32 and carried from token to token; what leaves is
// y_c silu(z_c), rounded once into the activations' type.
//
//   ia_selective_scan   the rows of the requests first_request .. first_request + B - 1 of a step, each from its state slot,
//                       which is left moved on.  A thread owns a channel with all its state values in registers; B and C of
//                       a token are the same for all channels and come from LDS, SEL_ROWS tokens at a time, every read
//                       one address for all lanes.  A request of more rows
//                       than `seg_len` is cut into segments of that many that run side by side: every segment but a
//                       request's last first runs from a zero state and leaves what it adds and the sum of its dt; a second
//                       kernel walks a request's segments, S <- exp(A sum dt) S + U, and leaves each the state before it;
//                       then every segment runs from that state and writes its rows, the last one the request's slot.
//
// The state lies [n][channel] in the slot, so that the lanes of a wave read and write neighbours.  All of it is fp32.
#include "common.h"

#define SEL_TB 4          // tokens whose channel values are asked for together
#define SEL_ROWS 32       // tokens whose B and C lie in LDS together (a multiple of SEL_TB)
#define SEL_BLOCK 128     // channels of a workgroup

// ln(1 + e^z) = max(z, 0) + ln(1 + w) with w = e^-|z| in (0, 1]; ln(1 + w) = 2 artanh(s), s = w / (2 + w) at most 1/3, by
// the series s + s^3/3 + ... + s^15/15 (the next term is below 5e-9 of the first): no difference of nearly equal
// numbers anywhere, so the result is good to a few units in the last place of fp32 for every z.
__device__ __forceinline__ float sel_softplus(float z) {
  const float w = __builtin_amdgcn_exp2f(-1.4426950408889634f * fabsf(z));
  const float s = w * __builtin_amdgcn_rcpf(2.0f + w), q = s * s;
  float p = 1.0f / 15.0f;
  p = __builtin_fmaf(p, q, 1.0f / 13.0f);
  p = __builtin_fmaf(p, q, 1.0f / 11.0f);
  p = __builtin_fmaf(p, q, 1.0f / 9.0f);
  p = __builtin_fmaf(p, q, 1.0f / 7.0f);
  p = __builtin_fmaf(p, q, 1.0f / 5.0f);
  p = __builtin_fmaf(p, q, 1.0f / 3.0f);
  p = __builtin_fmaf(p, q, 1.0f);
  return __builtin_fmaf(2.0f * s, p, fmaxf(z, 0.0f));
}

struct SelArgs {
  const float* dt_raw;           // rows of dt_stride values
  const float* dt_bias;          // [C]
  const float* a2;               // [Ns, C]: A log2(e)
  const float* skip;             // [C]
  float* state;
  long state_stride;
  const int* seq_starts;
  const int* state_slots;
  float* records;                // [segments of all requests, Ns, C]
  float* sums;                   // [segments of all requests, C]
  int dt_stride, x_stride, z_stride, bc_stride, b_col, c_col, out_stride, C, Ns, seg_len, first_request;
};

// The record of a request's first segment: the segments in the order of the requests.
__device__ __forceinline__ size_t sel_record(const SelArgs& P, int r) {
  int before = 0;
  for (int i = P.first_request; i < P.first_request + r; ++i)
    before += (P.seq_starts[i + 1] - P.seq_starts[i] + P.seg_len - 1) / P.seg_len;
  return (size_t)before;
}

// grid (blocks of SEL_BLOCK channels, segments, requests), SEL_BLOCK threads.  KN: state values a thread holds, Ns of them
// real (B and C have KN columns, those past Ns zero).  MODE 0: a request's rows from its slot; 1: what a segment adds; 2: a
// segment's rows.
template <typename T, int KN, int MODE>
__global__ __launch_bounds__(SEL_BLOCK) void selective_scan_kernel(const T* __restrict__ x, const T* __restrict__ z,
                                                                   const T* __restrict__ bc, T* __restrict__ out, SelArgs P) {
  constexpr int BC = MODE == 1 ? KN : 2 * KN;                    // floats of a token in LDS: B, and C where rows are written
  __shared__ __attribute__((aligned(16))) float s_bc[SEL_ROWS][BC];
  const int r = blockIdx.z, s = P.first_request + r, seg = blockIdx.y, tid = threadIdx.x;
  const int c = blockIdx.x * SEL_BLOCK + tid;
  int first = P.seq_starts[s], count = P.seq_starts[s + 1] - first;
  bool last = true;
  if (MODE != 0) {
    const int r0 = seg * P.seg_len;
    if (r0 >= count) return;
    last = r0 + P.seg_len >= count;
    if (MODE == 1 && last) return;
    first += r0;
    count = last ? count - r0 : P.seg_len;
  }
  if (count <= 0) return;
  const bool live = c < P.C;
  const int cc = live ? c : P.C - 1;
  const size_t rec = MODE == 0 ? 0 : sel_record(P, r) + seg;
  float* slot = P.state + (size_t)P.state_slots[s] * P.state_stride;
  float* R = MODE == 0 ? slot : P.records + rec * ((size_t)P.Ns * P.C);
  const T* xp = x + (size_t)first * P.x_stride + cc;
  const T* zp = z + (size_t)first * P.z_stride + cc;
  const float* dp = P.dt_raw + (size_t)first * P.dt_stride + cc;
  float xn[SEL_TB], zn[SEL_TB], dn[SEL_TB];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int k = 0; k < SEL_TB; ++k) {
      const int t = t0 + k < count ? t0 + k : count - 1;
      xn[k] = to_float(xp[(size_t)t * P.x_stride]);
      if (MODE != 1) zn[k] = to_float(zp[(size_t)t * P.z_stride]);
      dn[k] = dp[(size_t)t * P.dt_stride];
    }
  };
  fetch(0);
  float S[KN], A[KN];
#pragma unroll
  for (int n = 0; n < KN; ++n) {
    A[n] = n < P.Ns ? P.a2[(size_t)n * P.C + cc] : 0.f;
    S[n] = (MODE != 1 && n < P.Ns) ? R[(size_t)n * P.C + cc] : 0.f;
  }
  const float bias = P.dt_bias[cc], D = MODE == 1 ? 0.f : P.skip[cc];
  float total = 0.f;
  for (int b0 = 0; b0 < count; b0 += SEL_ROWS) {
    const int nb = count - b0 < SEL_ROWS ? count - b0 : SEL_ROWS;
    __syncthreads();                                              // the tokens before are read to their end
    for (int i = tid; i < nb * BC; i += SEL_BLOCK) {
      const int t = i / BC, n = i - t * BC;
      s_bc[t][n] = to_float(bc[(size_t)(first + b0 + t) * P.bc_stride + (n < KN ? P.b_col + n : P.c_col + (n - KN))]);
    }
    __syncthreads();
    for (int t0 = 0; t0 < nb; t0 += SEL_TB) {
      float xv[SEL_TB], zv[SEL_TB], dt[SEL_TB];
#pragma unroll
      for (int k = 0; k < SEL_TB; ++k) {
        xv[k] = xn[k];
        if (MODE != 1) zv[k] = zn[k];
        dt[k] = sel_softplus(dn[k] + bias);
      }
      if (b0 + t0 + SEL_TB < count) fetch(b0 + t0 + SEL_TB);
#pragma unroll
      for (int k = 0; k < SEL_TB; ++k) {
        if (t0 + k >= nb) break;                                   // the same for all lanes
        const float4* bt = reinterpret_cast<const float4*>(&s_bc[t0 + k][0]);
        const float d = dt[k], dx = d * xv[k];
        float y0 = 0.f, y1 = 0.f;
#pragma unroll
        for (int n = 0; n < KN; n += 4) {
          const float4 bv = bt[n / 4];
          S[n] = __builtin_fmaf(__builtin_amdgcn_exp2f(d * A[n]), S[n], dx * bv.x);
          S[n + 1] = __builtin_fmaf(__builtin_amdgcn_exp2f(d * A[n + 1]), S[n + 1], dx * bv.y);
          S[n + 2] = __builtin_fmaf(__builtin_amdgcn_exp2f(d * A[n + 2]), S[n + 2], dx * bv.z);
          S[n + 3] = __builtin_fmaf(__builtin_amdgcn_exp2f(d * A[n + 3]), S[n + 3], dx * bv.w);
          if (MODE != 1) {
            const float4 cv = bt[(KN + n) / 4];
            y0 = __builtin_fmaf(S[n], cv.x, y0);
            y1 = __builtin_fmaf(S[n + 1], cv.y, y1);
            y0 = __builtin_fmaf(S[n + 2], cv.z, y0);
            y1 = __builtin_fmaf(S[n + 3], cv.w, y1);
          }
        }
        if (MODE == 1) {
          total += d;
        } else if (live) {
          const float y = __builtin_fmaf(D, xv[k], y0 + y1), zz = zv[k];
          const float gate = zz * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * zz));
          out[(size_t)(first + b0 + t0 + k) * P.out_stride + c] = from_float<T>(y * gate);
        }
      }
    }
  }
  if (!live || (MODE == 2 && !last)) return;
  float* W = MODE == 1 ? R : slot;
#pragma unroll
  for (int n = 0; n < KN; ++n)
    if (n < P.Ns) W[(size_t)n * P.C + c] = S[n];
  if (MODE == 1) P.sums[rec * P.C + c] = total;
}

// grid (blocks of 256 of the state's values, requests): the record of a segment holds what the segment adds when a thread
// comes and the state before the segment when it goes.  Four segments' loads are in flight together.
#define SEL_AHEAD 4
__global__ __launch_bounds__(256) void selective_chain_kernel(SelArgs P) {
  const int r = blockIdx.y, s = P.first_request + r;
  const int e = blockIdx.x * 256 + threadIdx.x;
  const int size = P.Ns * P.C;
  if (e >= size) return;
  const int rows = P.seq_starts[s + 1] - P.seq_starts[s];
  const int count = (rows + P.seg_len - 1) / P.seg_len;
  const int c = e % P.C;
  const float a = P.a2[e];
  float S = P.state[(size_t)P.state_slots[s] * P.state_stride + e];
  const size_t rec = sel_record(P, r);
  float* R = P.records + rec * size + e;
  const float* Q = P.sums + rec * P.C + c;
  for (int j0 = 0; j0 < count; j0 += SEL_AHEAD) {
    float U[SEL_AHEAD], T[SEL_AHEAD];
#pragma unroll
    for (int k = 0; k < SEL_AHEAD; ++k) {
      const bool adds = j0 + k < count - 1;                   // a request's last segment adds nothing that anyone reads
      U[k] = adds ? R[(size_t)(j0 + k) * size] : 0.f;
      T[k] = adds ? Q[(size_t)(j0 + k) * P.C] : 0.f;
    }
#pragma unroll
    for (int k = 0; k < SEL_AHEAD; ++k) {
      if (j0 + k >= count) break;
      R[(size_t)(j0 + k) * size] = S;
      if (j0 + k < count - 1) S = __builtin_fmaf(exp2f(a * T[k]), S, U[k]);
    }
  }
}

// The state values a thread holds for Ns real ones: B and C need so many columns each.  0: more than the kernel takes.
extern "C" int ia_selective_columns(int Ns) {
  for (int k = 8; k <= 128; k *= 2)
    if (Ns <= k) return k;
  return 0;
}

// x, z, bc: rows of the activations' type (code): the channels behind their convolution, the gates' logits, and a row that
// holds ia_selective_columns(Ns) values of B from b_col and as many of C from c_col (values past Ns
// zero).  dt_raw fp32.  a2 fp32 [Ns, C]: A log2(e).  out: rows of out_stride values.  max_rows: at least the rows of
// the longest of the requests; with more than seg_len: records fp32 [segments, Ns, C] and sums [segments, C] for the
// segments of all requests (ceil(rows / seg_len) each).
extern "C" int ia_selective_scan(const void* x, int code, int x_stride, const void* z, int z_stride, const void* bc,
                                 int bc_stride, int b_col, int c_col, const float* dt_raw, int dt_stride,
                                 const float* dt_bias, const float* a2, const float* skip, float* state, long state_stride,
                                 void* out, int out_stride, const int* seq_starts, const int* state_slots, int first_request,
                                 int B, int C, int Ns, int max_rows, int seg_len, float* records, float* sums,
                                 hipStream_t stream) {
  if (B == 0) return IA_OK;
  if (!x || !z || !bc || !dt_raw || !dt_bias || !a2 || !skip || !state || !out || !seq_starts || !state_slots || B < 0 ||
      B > 65535 || C <= 0 || Ns <= 0 || first_request < 0 || max_rows <= 0 || seg_len <= 0 || x_stride < C || z_stride < C ||
      dt_stride < C || out_stride < C || state_stride < (long)Ns * C)
    return IA_ERR_BAD_ARG;
  const int kn = ia_selective_columns(Ns);
  if (kn == 0) return IA_ERR_UNSUPPORTED;
  if (b_col < 0 || c_col < 0 || bc_stride < b_col + kn || bc_stride < c_col + kn) return IA_ERR_BAD_ARG;
  const int segs = (max_rows + seg_len - 1) / seg_len;
  if (segs > 65535) return IA_ERR_UNSUPPORTED;
  if (segs > 1 && (!records || !sums)) return IA_ERR_BAD_ARG;
  const SelArgs P{dt_raw, dt_bias, a2, skip, state, state_stride, seq_starts, state_slots, records, sums,
                  dt_stride, x_stride, z_stride, bc_stride, b_col, c_col, out_stride, C, Ns, seg_len, first_request};
  const unsigned blocks = (unsigned)((C + SEL_BLOCK - 1) / SEL_BLOCK);
#define IA_SEL(T, KN, MODE, SEGS)                                                                                     \
  selective_scan_kernel<T, KN, MODE><<<dim3(blocks, (unsigned)(SEGS), (unsigned)B), SEL_BLOCK, 0, stream>>>(            \
      (const T*)x, (const T*)z, (const T*)bc, (T*)out, P)
#define IA_SEL_K(T, MODE, SEGS)                   \
  do {                                            \
    if (kn == 8) IA_SEL(T, 8, MODE, SEGS);        \
    else if (kn == 16) IA_SEL(T, 16, MODE, SEGS); \
    else if (kn == 32) IA_SEL(T, 32, MODE, SEGS); \
    else if (kn == 64) IA_SEL(T, 64, MODE, SEGS); \
    else IA_SEL(T, 128, MODE, SEGS);              \
  } while (0)
#define IA_SEL_T(MODE, SEGS)                        \
  do {                                              \
    if (code == IA_F32) IA_SEL_K(float, MODE, SEGS); \
    else IA_SEL_K(bf16_t, MODE, SEGS);              \
  } while (0)
  if (code != IA_F32 && code != IA_BF16) return IA_ERR_BAD_ARG;
  if (segs == 1) {
    IA_SEL_T(0, 1);
    IA_LAUNCH_CHECK();
    return IA_OK;
  }
  IA_SEL_T(1, segs);
  IA_LAUNCH_CHECK();
  selective_chain_kernel<<<dim3((unsigned)(((long)Ns * C + 255) / 256), (unsigned)B), 256, 0, stream>>>(P);
  IA_LAUNCH_CHECK();
  IA_SEL_T(2, segs);
#undef IA_SEL_T
#undef IA_SEL_K
#undef IA_SEL
  IA_LAUNCH_CHECK();
  return IA_OK;
}

#include "op_call.h"
IA_OP(ia_selective_scan)
