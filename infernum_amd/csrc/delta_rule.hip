// The generalized delta rule: a recurrence per head over a state S [dim, dim] of fp32 values in which every token
// decays the state channel by channel, takes out part of what lies along its key, and writes its own key and value:
//
//     S_t = diag(w_t) S_(t-1) - (a_t * u_t) (u_t^T S_(t-1)) + k_t v_t^T,        o_t = S_t^T r_t,
//
// with u = k / sqrt(sum k^2 + eps) the head's unit key, w = exp(-c sigmoid(z + w0)) the decay of every key channel and
// a = sigmoid(za + ab) how much of what u finds in the state is taken out.  Both terms read the old state.
//
//   ia_delta_tanh_rows   the middle of the decay logits' two products: tanh of some columns of the projected rows.
//   ia_delta_prepare     per token and head: z <- w in place, a, and 1 / sqrt(sum k^2 + eps); all fp32.
//   ia_delta_scan        the recurrence token after token for the rows of every request of a step, from the request's
//                        state slot, which it leaves moved on.
//
// A column of S needs nothing of the other columns, so a wave takes four columns: sixteen lanes share a column's
// channels (in registers, a lane dim / 16 of them), the sums over the channels are four rotations within the sixteen
// lanes (every lane ends with the same bits), and a token costs no barrier and no trip through LDS but the reads of
// the token's vectors, which DR_WAVES waves of a workgroup bring into LDS together, DR_TB tokens at a time, the next
// ones' loads in flight meanwhile.  The chain of operations of a column is the same however the tokens are cut into
// steps and whatever else the step holds.
//
// A head's state is kept column by column: slot[head][column][channel].
#include "common.h"

#define DR_TB 8          // tokens whose vectors are staged together
#define DR_WAVES 2       // waves of a workgroup: 8 columns
#define DR_COLS (4 * DR_WAVES)

// Sum over the sixteen lanes of a row of lanes, the same bits in every lane (each step adds two numbers that the
// other lane of the pair adds too).
__device__ __forceinline__ float dr_sum16(float x) {
#define DR_ROR(n) x += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), 0x120 + (n), 0xf, 0xf, true))
  DR_ROR(8);
  DR_ROR(4);
  DR_ROR(2);
  DR_ROR(1);
#undef DR_ROR
  return x;
}

template <typename T>
__global__ __launch_bounds__(256) void delta_tanh_rows_kernel(const T* __restrict__ src, int src_stride, T* __restrict__ dst,
                                                              long total, int C) {
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const long n = i / C;
  const int c = (int)(i - n * C);
  dst[i] = from_float<T>(tanhf(to_float(src[(size_t)n * src_stride + c])));
}

extern "C" int ia_delta_tanh_rows(const void* src, int src_stride, void* dst, int dtype, int N, int C, hipStream_t stream) {
  if (N < 0 || C <= 0 || src_stride < C || (dtype != IA_F32 && dtype != IA_BF16)) return IA_ERR_BAD_ARG;
  if (N == 0) return IA_OK;
  if (!src || !dst) return IA_ERR_BAD_ARG;
  const long total = (long)N * C;
  const unsigned grid = (unsigned)((total + 255) / 256);
  if (dtype == IA_F32) delta_tanh_rows_kernel<float><<<grid, 256, 0, stream>>>((const float*)src, src_stride, (float*)dst, total, C);
  else delta_tanh_rows_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)src, src_stride, (bf16_t*)dst, total, C);
  IA_LAUNCH_CHECK();
  return IA_OK;
}

// A wave a (token, head).  k and za: columns of the projected rows.
template <typename T>
__global__ __launch_bounds__(256) void delta_prepare_kernel(const T* __restrict__ proj, int proj_stride, int k_col, int a_col,
                                                            float* __restrict__ z, const float* __restrict__ w0,
                                                            const float* __restrict__ ab, float* __restrict__ a,
                                                            float* __restrict__ inv, long pairs, int nh, int dim,
                                                            float decay_scale, float eps) {
  const long pair = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (pair >= pairs) return;
  const int lane = threadIdx.x & 63;
  const long n = pair / nh;
  const int hd = (int)(pair - n * nh);
  const T* row = proj + (size_t)n * proj_stride;
  const size_t at = (size_t)pair * dim;
  float ss = 0.f;
  for (int i = lane; i < dim; i += 64) {
    const int c = hd * dim + i;
    const float k = to_float(row[k_col + c]);
    ss = __builtin_fmaf(k, k, ss);
    const float zz = z[at + i] + w0[c];
    z[at + i] = expf(-decay_scale * (1.0f / (1.0f + expf(-zz))));
    a[at + i] = 1.0f / (1.0f + expf(-(to_float(row[a_col + c]) + ab[c])));
  }
  ss = wave_sum(ss);
  if (lane == 0) inv[pair] = 1.0f / sqrtf(ss + eps);
}

extern "C" int ia_delta_prepare(const void* proj, int code, int proj_stride, int k_col, int a_col, float* z, const float* w0,
                                const float* ab, float* a, float* inv, int N, int nh, int dim, float decay_scale, float eps,
                                hipStream_t stream) {
  if (N < 0 || nh <= 0 || dim <= 0 || k_col < 0 || a_col < 0 || proj_stride < k_col + nh * dim ||
      proj_stride < a_col + nh * dim || (code != IA_F32 && code != IA_BF16))
    return IA_ERR_BAD_ARG;
  if (N == 0) return IA_OK;
  if (!proj || !z || !w0 || !ab || !a || !inv) return IA_ERR_BAD_ARG;
  const long pairs = (long)N * nh;
  const unsigned grid = (unsigned)((pairs + 3) / 4);
  if (code == IA_F32)
    delta_prepare_kernel<float><<<grid, 256, 0, stream>>>((const float*)proj, proj_stride, k_col, a_col, z, w0, ab, a, inv,
                                                          pairs, nh, dim, decay_scale, eps);
  else
    delta_prepare_kernel<bf16_t><<<grid, 256, 0, stream>>>((const bf16_t*)proj, proj_stride, k_col, a_col, z, w0, ab, a, inv,
                                                           pairs, nh, dim, decay_scale, eps);
  IA_LAUNCH_CHECK();
  return IA_OK;
}

// VEC channels side by side a lane and J such groups, 16 VEC apart: lane q holds the channels 16 VEC j + VEC q + e.
// Channels past the head's last are zero everywhere and stay zero.
template <int VEC>
__device__ __forceinline__ void dr_read(const float* p, float (&v)[VEC]) {
  if (VEC == 4) {
    const float4 t = *reinterpret_cast<const float4*>(p);
    v[0] = t.x;
    v[1 % VEC] = t.y;
    v[2 % VEC] = t.z;
    v[3 % VEC] = t.w;
  } else if (VEC == 2) {
    const float2 t = *reinterpret_cast<const float2*>(p);
    v[0] = t.x;
    v[1 % VEC] = t.y;
  } else {
    v[0] = p[0];
  }
}

// A barrier for what goes through LDS alone: __syncthreads() would also wait for the results' stores on their way to
// memory, which no other thread reads.
__device__ __forceinline__ void dr_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}

// The vectors of one token as a lane needs them.
template <int VEC, int J>
struct DrToken {
  float u[J][VEC], w[J][VEC], au[J][VEC], k[J][VEC], r[J][VEC], v;
};

// L values side by side from memory, as they are stored there (converted when they go to LDS: nothing waits here).
template <typename T, int L> struct DrRaw;
template <> struct DrRaw<float, 1> { typedef float type; };
template <> struct DrRaw<float, 4> { typedef float4 type; };
template <> struct DrRaw<bf16_t, 1> { typedef bf16_t type; };
template <> struct DrRaw<bf16_t, 4> { typedef uint2 type; };
__device__ __forceinline__ void dr_values(float x, float (&o)[1]) { o[0] = x; }
__device__ __forceinline__ void dr_values(bf16_t x, float (&o)[1]) { o[0] = to_float(x); }
__device__ __forceinline__ void dr_values(float4 x, float (&o)[4]) { o[0] = x.x; o[1] = x.y; o[2] = x.z; o[3] = x.w; }
__device__ __forceinline__ void dr_values(uint2 x, float (&o)[4]) {
  o[0] = __uint_as_float(x.x << 16);
  o[1] = __uint_as_float(x.x & 0xffff0000u);
  o[2] = __uint_as_float(x.y << 16);
  o[3] = __uint_as_float(x.y & 0xffff0000u);
}
__device__ __forceinline__ void dr_put(float* at, const float (&v)[1]) { at[0] = v[0]; }
__device__ __forceinline__ void dr_put(float* at, const float (&v)[4]) {
  *reinterpret_cast<float4*>(at) = make_float4(v[0], v[1], v[2], v[3]);
}

// grid (heads, requests, groups of DR_COLS columns), 64 DR_WAVES threads.  L: channels of a load when vectors are staged
// (4 where every row and column begins on a multiple of four values, else 1).
template <typename T, int VEC, int J, int L>
__global__ __launch_bounds__(64 * DR_WAVES) void delta_scan_kernel(
    const T* __restrict__ proj, int proj_stride, int r_col, int k_col, int v_col, const float* __restrict__ w,
    const float* __restrict__ a, const float* __restrict__ inv, float* __restrict__ state, long state_stride,
    float* __restrict__ out, const int* __restrict__ seq_starts, const int* __restrict__ state_slots, int nh, int dim) {
  constexpr int P = 16 * VEC * J;                     // the channels with those that pad them
  constexpr int NT = 64 * DR_WAVES;
  constexpr int PER = (DR_TB * P / L + NT - 1) / NT;  // pieces of L channels a thread stages, of each vector
  static_assert(P % L == 0 && DR_TB * DR_COLS <= NT, "pieces fit the rows; a thread stages at most one value of v");
  __shared__ __attribute__((aligned(16))) float s_w[DR_TB][P], s_au[DR_TB][P], s_u[DR_TB][P], s_k[DR_TB][P], s_r[DR_TB][P];
  __shared__ float s_v[DR_TB][DR_COLS];
  const int hd = blockIdx.x, s = blockIdx.y, c0 = blockIdx.z * DR_COLS;
  const int first = seq_starts[s], count = seq_starts[s + 1] - first;
  if (count <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, q = lane & 15, grp = wave * 4 + (lane >> 4);
  const int col = c0 + grp;                           // this lane's column of the state
  const bool col_ok = col < dim;
  float* st = state + (size_t)state_slots[s] * state_stride + ((size_t)hd * dim + (col_ok ? col : 0)) * dim;
  // the vectors of up to DR_TB tokens on their way to LDS: every load is made, from a place of this head's own rows where
  // there is no such token or channel (those values are replaced by zeros on the way into LDS)
  typename DrRaw<float, L>::type fw[PER], fa[PER];
  typename DrRaw<T, L>::type fk[PER], fr[PER];
  float fi[PER];
  T fv;
  auto fetch = [&](int t0) {
#pragma unroll
    for (int x = 0; x < PER; ++x) {
      const int idx = tid + x * NT, t = idx / (P / L), n = (idx - t * (P / L)) * L;
      const int tc = t0 + t < count ? t0 + t : count - 1, nc = n < dim ? n : 0;
      const size_t row = (size_t)(first + tc), at = (row * nh + hd) * dim + nc;
      const T* pr = proj + row * proj_stride + hd * dim + nc;
      fw[x] = *reinterpret_cast<const typename DrRaw<float, L>::type*>(w + at);
      fa[x] = *reinterpret_cast<const typename DrRaw<float, L>::type*>(a + at);
      fk[x] = *reinterpret_cast<const typename DrRaw<T, L>::type*>(pr + k_col);
      fr[x] = *reinterpret_cast<const typename DrRaw<T, L>::type*>(pr + r_col);
      fi[x] = inv[row * nh + hd];
    }
    const int t = tid / DR_COLS, c = c0 + tid % DR_COLS;
    fv = proj[(size_t)(first + (t0 + t < count ? t0 + t : count - 1)) * proj_stride + v_col + hd * dim + (c < dim ? c : 0)];
  };
  float S[J][VEC];
#pragma unroll
  for (int j = 0; j < J; ++j)
#pragma unroll
    for (int e = 0; e < VEC; ++e) S[j][e] = 0.f;
#pragma unroll
  for (int j = 0; j < J; ++j) {
    const int n = 16 * VEC * j + VEC * q;
    if (VEC == L && L == 4) {                         // channels in fours: all of them are there or none
      if (col_ok && n < dim) dr_read<VEC>(st + n, S[j]);
    } else {
#pragma unroll
      for (int e = 0; e < VEC; ++e)
        if (col_ok && n + e < dim) S[j][e] = st[n + e];
    }
  }
  fetch(0);
  // the state is in its registers from here on: a use of it inside the loop must not be taken for one that waits for a
  // load, which would make every turn wait for the next tokens' vectors as well
#pragma unroll
  for (int j = 0; j < J; ++j)
#pragma unroll
    for (int e = 0; e < VEC; ++e) asm volatile("" : "+v"(S[j][e]));
  DrToken<VEC, J> A, B;
  auto load = [&](int t, DrToken<VEC, J>& X) {
#pragma unroll
    for (int j = 0; j < J; ++j) {
      const int n = 16 * VEC * j + VEC * q;
      dr_read<VEC>(&s_u[t][n], X.u[j]);
      dr_read<VEC>(&s_w[t][n], X.w[j]);
      dr_read<VEC>(&s_au[t][n], X.au[j]);
      dr_read<VEC>(&s_k[t][n], X.k[j]);
      dr_read<VEC>(&s_r[t][n], X.r[j]);
    }
    X.v = s_v[t][grp];
  };
  auto step = [&](const DrToken<VEC, J>& X) {
    float d[J];
#pragma unroll
    for (int j = 0; j < J; ++j) {
      d[j] = X.u[j][0] * S[j][0];
#pragma unroll
      for (int e = 1; e < VEC; ++e) d[j] = __builtin_fmaf(X.u[j][e], S[j][e], d[j]);
    }
#pragma unroll
    for (int j = 1; j < J; ++j) d[0] += d[j];
    const float dot = dr_sum16(d[0]);                 // u^T S of this column
    float o[J];
#pragma unroll
    for (int j = 0; j < J; ++j) {
      o[j] = 0.f;
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        const float add = __builtin_fmaf(X.k[j][e], X.v, -(X.au[j][e] * dot));
        S[j][e] = __builtin_fmaf(X.w[j][e], S[j][e], add);
        o[j] = __builtin_fmaf(X.r[j][e], S[j][e], o[j]);
      }
    }
#pragma unroll
    for (int j = 1; j < J; ++j) o[0] += o[j];
    return dr_sum16(o[0]);
  };
  for (int t0 = 0; t0 < count; t0 += DR_TB) {
    const int nt = count - t0 < DR_TB ? count - t0 : DR_TB;
    dr_barrier();                                     // the tokens before are read to their end
#pragma unroll
    for (int x = 0; x < PER; ++x) {
      const int idx = tid + x * NT, t = idx / (P / L), n = (idx - t * (P / L)) * L;
      float vw[L], va[L], vk[L], vr[L], u[L];
      dr_values(fw[x], vw);
      dr_values(fa[x], va);
      dr_values(fk[x], vk);
      dr_values(fr[x], vr);
      const bool real = n < dim && t < nt;
#pragma unroll
      for (int e = 0; e < L; ++e) {
        u[e] = real ? vk[e] * fi[x] : 0.f;
        va[e] = real ? va[e] * u[e] : 0.f;
        vw[e] = real ? vw[e] : 0.f;
        vk[e] = real ? vk[e] : 0.f;
        vr[e] = real ? vr[e] : 0.f;
      }
      if (t < DR_TB) {
        dr_put(&s_w[t][n], vw);
        dr_put(&s_au[t][n], va);
        dr_put(&s_u[t][n], u);
        dr_put(&s_k[t][n], vk);
        dr_put(&s_r[t][n], vr);
      }
    }
    if (tid < DR_TB * DR_COLS) s_v[tid / DR_COLS][tid % DR_COLS] = c0 + tid % DR_COLS < dim ? to_float(fv) : 0.f;
    dr_barrier();
    if (t0 + DR_TB < count) fetch(t0 + DR_TB);
    float mine = 0.f;                                 // lane q keeps token q's result of the column
    load(0, A);
    if (nt == DR_TB) {                                // the next token's vectors come in while this one is worked on
#pragma unroll
      for (int t = 0; t < DR_TB; t += 2) {
        load(t + 1, B);
        const float o0 = step(A);
        mine = q == t ? o0 : mine;
        if (t + 2 < DR_TB) load(t + 2, A);
        const float o1 = step(B);
        mine = q == t + 1 ? o1 : mine;
      }
    } else {
      for (int t = 0; t < nt; ++t) {
        const float o = step(A);
        mine = q == t ? o : mine;
        if (t + 1 < nt) load(t + 1, A);
      }
    }
    if (col_ok && q < nt) out[((size_t)(first + t0 + q) * nh + hd) * dim + col] = mine;
  }
#pragma unroll
  for (int j = 0; j < J; ++j) {
    const int n = 16 * VEC * j + VEC * q;
    if (VEC == L && L == 4) {
      if (col_ok && n < dim) *reinterpret_cast<float4*>(st + n) = make_float4(S[j][0], S[j][1 % VEC], S[j][2 % VEC], S[j][3 % VEC]);
    } else {
#pragma unroll
      for (int e = 0; e < VEC; ++e)
        if (col_ok && n + e < dim) st[n + e] = S[j][e];
    }
  }
}

// Floats a request's slot holds for one layer run.
extern "C" long ia_delta_state_floats(int nh, int dim) { return (long)nh * dim * dim; }

// proj: rows of proj_stride values (code: their type) holding r, k and v (nh dim values each from their columns); w, a
// fp32 [N, nh, dim] and inv fp32 [N, nh] as ia_delta_prepare leaves them; out fp32 [N, nh, dim].
extern "C" int ia_delta_scan(const void* proj, int code, int proj_stride, int r_col, int k_col, int v_col, const float* w,
                             const float* a, const float* inv, float* state, long state_stride, float* out,
                             const int* seq_starts, const int* state_slots, int B, int nh, int dim, hipStream_t stream) {
  if (B == 0) return IA_OK;
  if (!proj || !w || !a || !inv || !state || !out || !seq_starts || !state_slots || B < 0 || nh <= 0 || dim <= 0 ||
      r_col < 0 || k_col < 0 || v_col < 0 || proj_stride < r_col + nh * dim || proj_stride < k_col + nh * dim ||
      proj_stride < v_col + nh * dim || state_stride < ia_delta_state_floats(nh, dim) || (code != IA_F32 && code != IA_BF16))
    return IA_ERR_BAD_ARG;
  const int groups = (dim + DR_COLS - 1) / DR_COLS;
  if (dim > 256 || B > 65535 || groups > 65535) return IA_ERR_UNSUPPORTED;
  const dim3 grid((unsigned)nh, (unsigned)B, (unsigned)groups);
  // in fours where every address that a piece of four values is read from is a multiple of its size
  const size_t el = code == IA_F32 ? 4 : 2;
  const bool fours = ((dim | proj_stride | r_col | k_col) & 3) == 0 && ((uintptr_t)proj % (4 * el)) == 0 && (state_stride & 3) == 0 &&
                     (((uintptr_t)w | (uintptr_t)a | (uintptr_t)state) & 15) == 0;
#define IA_DR(T, V, JJ)                                                                                                    \
  do {                                                                                                                     \
    if (fours)                                                                                                             \
      delta_scan_kernel<T, V, JJ, 4><<<grid, 64 * DR_WAVES, 0, stream>>>((const T*)proj, proj_stride, r_col, k_col, v_col, \
                                                                         w, a, inv, state, state_stride, out, seq_starts,  \
                                                                         state_slots, nh, dim);                            \
    else                                                                                                                   \
      delta_scan_kernel<T, V, JJ, 1><<<grid, 64 * DR_WAVES, 0, stream>>>((const T*)proj, proj_stride, r_col, k_col, v_col, \
                                                                         w, a, inv, state, state_stride, out, seq_starts,  \
                                                                         state_slots, nh, dim);                            \
  } while (0)
#define IA_DR_D(T)                         \
  do {                                     \
    if (dim <= 16) IA_DR(T, 1, 1);         \
    else if (dim <= 32) IA_DR(T, 2, 1);    \
    else if (dim <= 64) IA_DR(T, 4, 1);    \
    else if (dim <= 96) IA_DR(T, 2, 3);    \
    else if (dim <= 128) IA_DR(T, 4, 2);   \
    else if (dim <= 192) IA_DR(T, 4, 3);   \
    else IA_DR(T, 4, 4);                   \
  } while (0)
  if (code == IA_F32) IA_DR_D(float);
  else IA_DR_D(bf16_t);
#undef IA_DR_D
#undef IA_DR
  IA_LAUNCH_CHECK();
  return IA_OK;
}

#include "op_call.h"
IA_OP(ia_delta_tanh_rows)
IA_OP(ia_delta_prepare)
IA_OP(ia_delta_scan)
