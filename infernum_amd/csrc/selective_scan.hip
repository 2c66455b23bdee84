// The selective scan with a decay per channel and state value (the Mamba-1 form):
//
//     dt = softplus(raw + bias_c),      S[n] <- exp(dt A[c, n]) S[n] + dt x_c B[n],      y_c = sum_n S[n] C[n] + D_c x_c,
//
// B and C shared by all channels of a token, the state fp32 and carried from token to token; what leaves is
// y_c silu(z_c), rounded once into the activations' type.
//
//   ia_selective_scan   the rows of the requests first_request .. first_request + B - 1 of a step, each from its state slot,
//                       which is left moved on.  A thread owns a channel with all its state values in registers; B and C of
//                       a token are the same for all lanes of a wave and come through scalar loads.  A request of more rows
//                       than `seg_len` is cut into segments of that many that run side by side: every segment but a
//                       request's last first runs from a zero state and leaves what it adds and the sum of its dt; a second
//                       kernel walks a request's segments, S <- exp(A sum dt) S + U, and leaves each the state before it;
//                       then every segment runs from that state and writes its rows, the last one the request's slot.
//
// The state lies [n][channel] in the slot, so that the lanes of a wave read and write neighbours.  All of it is fp32.
#include "common.h"

#define SEL_TB 4          // tokens whose channel values are asked for together

__device__ __forceinline__ float sel_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// Two neighbouring values of a row that is the same for all lanes.
template <typename T> struct SelPair;
template <> struct SelPair<bf16_t> {
  static __device__ __forceinline__ void get(const bf16_t* p, int i, float& a, float& b) {
    const uint32_t w = reinterpret_cast<const uint32_t*>(p)[i];
    a = __uint_as_float(w << 16);
    b = __uint_as_float(w & 0xffff0000u);
  }
};
template <> struct SelPair<float> {
  static __device__ __forceinline__ void get(const float* p, int i, float& a, float& b) {
    a = p[2 * i];
    b = p[2 * i + 1];
  }
};

struct SelArgs {
  const float* dt_raw;           // rows of dt_stride values
  const float* dt_bias;          // [C]
  const float* a2;               // [Ns, C]: A log2(e)
  const float* skip;             // [C]
  float* state;
  long state_stride;
  const int* seq_starts;
  const int* state_slots;
  float* records;                // [requests, max_segs, Ns, C]
  float* sums;                   // [requests, max_segs, C]
  int dt_stride, x_stride, z_stride, bc_stride, b_col, c_col, out_stride, C, Ns, seg_len, max_segs, first_request;
};

// grid (blocks of 64 channels, segments, requests), 64 threads.  KN: state values a thread holds, Ns of them real (B and C
// have KN columns, those past Ns zero).  MODE 0: a request's rows from its slot; 1: what a segment adds; 2: a segment's rows.
template <typename T, int KN, int MODE>
__global__ __launch_bounds__(64) void selective_scan_kernel(const T* __restrict__ x, const T* __restrict__ z,
                                                            const T* __restrict__ bc, T* __restrict__ out, SelArgs P) {
  const int r = blockIdx.z, s = P.first_request + r, seg = blockIdx.y;
  const int c = blockIdx.x * 64 + threadIdx.x;
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
  const size_t rec = (size_t)r * P.max_segs + seg;
  float* slot = P.state + (size_t)P.state_slots[s] * P.state_stride;
  float* R = MODE == 0 ? slot : P.records + rec * ((size_t)P.Ns * P.C);
  float S[KN], A[KN];
#pragma unroll
  for (int n = 0; n < KN; ++n) {
    A[n] = n < P.Ns ? P.a2[(size_t)n * P.C + cc] : 0.f;
    S[n] = (MODE != 1 && n < P.Ns) ? R[(size_t)n * P.C + cc] : 0.f;
  }
  const float bias = P.dt_bias[cc], D = MODE == 1 ? 0.f : P.skip[cc];
  float total = 0.f;
  float xn[SEL_TB], zn[SEL_TB], dn[SEL_TB];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int k = 0; k < SEL_TB; ++k) {
      const int t = t0 + k < count ? t0 + k : count - 1;
      const size_t row = (size_t)(first + t);
      xn[k] = to_float(x[row * P.x_stride + cc]);
      if (MODE != 1) zn[k] = to_float(z[row * P.z_stride + cc]);
      dn[k] = P.dt_raw[row * P.dt_stride + cc];
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < count; t0 += SEL_TB) {
    float xv[SEL_TB], zv[SEL_TB], dt[SEL_TB];
#pragma unroll
    for (int k = 0; k < SEL_TB; ++k) {
      xv[k] = xn[k];
      if (MODE != 1) zv[k] = zn[k];
      dt[k] = sel_softplus(dn[k] + bias);
    }
    if (t0 + SEL_TB < count) fetch(t0 + SEL_TB);
#pragma unroll
    for (int k = 0; k < SEL_TB; ++k) {
      if (t0 + k >= count) break;                                  // the same for all lanes
      const T* br = bc + (size_t)(first + t0 + k) * P.bc_stride + P.b_col;
      const T* cr = bc + (size_t)(first + t0 + k) * P.bc_stride + P.c_col;
      const float d = dt[k], dx = d * xv[k];
      float y0 = 0.f, y1 = 0.f;
#pragma unroll
      for (int n = 0; n < KN; n += 2) {
        float b0, b1, c0, c1;
        SelPair<T>::get(br, n / 2, b0, b1);
        S[n] = __builtin_fmaf(__builtin_amdgcn_exp2f(d * A[n]), S[n], dx * b0);
        S[n + 1] = __builtin_fmaf(__builtin_amdgcn_exp2f(d * A[n + 1]), S[n + 1], dx * b1);
        if (MODE != 1) {
          SelPair<T>::get(cr, n / 2, c0, c1);
          y0 = __builtin_fmaf(S[n], c0, y0);
          y1 = __builtin_fmaf(S[n + 1], c1, y1);
        }
      }
      if (MODE == 1) {
        total += d;
      } else if (live) {
        const float y = __builtin_fmaf(D, xv[k], y0 + y1);
        out[(size_t)(first + t0 + k) * P.out_stride + c] = from_float<T>(y * (zv[k] / (1.0f + expf(-zv[k]))));
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
  float* R = P.records + (size_t)r * P.max_segs * size + e;
  const float* Q = P.sums + (size_t)r * P.max_segs * P.C + c;
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
// holds ia_selective_columns(Ns) values of B from b_col and as many of C from c_col (even columns, even bc_stride; values
// past Ns zero).  dt_raw fp32.  a2 fp32 [Ns, C]: A log2(e).  out: rows of out_stride values.  max_rows: at least the rows of
// the longest of the requests; with more than seg_len: records fp32 [B, ceil(max_rows / seg_len), Ns, C] and sums
// [B, ceil(max_rows / seg_len), C].
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
  if ((b_col | c_col | bc_stride) & 1 || ((uintptr_t)bc & 3)) return IA_ERR_UNSUPPORTED;
  const int segs = (max_rows + seg_len - 1) / seg_len;
  if (segs > 65535) return IA_ERR_UNSUPPORTED;
  if (segs > 1 && (!records || !sums)) return IA_ERR_BAD_ARG;
  const SelArgs P{dt_raw, dt_bias, a2, skip, state, state_stride, seq_starts, state_slots, records, sums,
                  dt_stride, x_stride, z_stride, bc_stride, b_col, c_col, out_stride, C, Ns, seg_len, segs, first_request};
  const unsigned blocks = (unsigned)((C + 63) / 64);
#define IA_SEL(T, KN, MODE, SEGS)                                                                                     \
  selective_scan_kernel<T, KN, MODE><<<dim3(blocks, (unsigned)(SEGS), (unsigned)B), 64, 0, stream>>>(                   \
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
