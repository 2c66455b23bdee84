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

// grid (heads, requests, groups of DR_COLS columns), 64 DR_WAVES threads.
template <typename T, int VEC, int J>
__global__ __launch_bounds__(64 * DR_WAVES) void delta_scan_kernel(
    const T* __restrict__ proj, int proj_stride, int r_col, int k_col, int v_col, const float* __restrict__ w,
    const float* __restrict__ a, const float* __restrict__ inv, float* __restrict__ state, long state_stride,
    float* __restrict__ out, const int* __restrict__ seq_starts, const int* __restrict__ state_slots, int nh, int dim) {
  constexpr int P = 16 * VEC * J;                     // the channels with those that pad them
  constexpr int NT = 64 * DR_WAVES;
  constexpr int PER = (DR_TB * P + NT - 1) / NT;      // channel values a thread stages, of each vector
  __shared__ __attribute__((aligned(16))) float s_w[DR_TB][P], s_au[DR_TB][P], s_u[DR_TB][P], s_k[DR_TB][P], s_r[DR_TB][P];
  __shared__ float s_v[DR_TB][DR_COLS];
  const int hd = blockIdx.x, s = blockIdx.y, c0 = blockIdx.z * DR_COLS;
  const int first = seq_starts[s], count = seq_starts[s + 1] - first;
  if (count <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, q = lane & 15, grp = wave * 4 + (lane >> 4);
  const int col = c0 + grp;                           // this lane's column of the state
  const bool col_ok = col < dim;
  float* st = state + (size_t)state_slots[s] * state_stride + ((size_t)hd * dim + (col_ok ? col : 0)) * dim;
  float S[J][VEC];
#pragma unroll
  for (int j = 0; j < J; ++j)
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      const int n = 16 * VEC * j + VEC * q + e;
      S[j][e] = (col_ok && n < dim) ? st[n] : 0.f;
    }
  // the vectors of up to DR_TB tokens on their way to LDS
  float fw[PER], fa[PER], fk[PER], fr[PER], fi[PER], fv = 0.f;
  auto fetch = [&](int t0) {
#pragma unroll
    for (int x = 0; x < PER; ++x) {
      const int idx = tid + x * NT, t = idx / P, n = idx - t * P;
      fw[x] = fa[x] = fk[x] = fr[x] = fi[x] = 0.f;
      if (t < DR_TB && t0 + t < count && n < dim) {
        const size_t row = (size_t)(first + t0 + t), at = (row * nh + hd) * dim + n;
        const T* pr = proj + row * proj_stride + hd * dim + n;
        fw[x] = w[at];
        fa[x] = a[at];
        fk[x] = to_float(pr[k_col]);
        fr[x] = to_float(pr[r_col]);
        fi[x] = inv[row * nh + hd];
      }
    }
    const int t = tid / DR_COLS, c = c0 + tid % DR_COLS;
    fv = 0.f;
    if (t < DR_TB && t0 + t < count && c < dim) fv = to_float(proj[(size_t)(first + t0 + t) * proj_stride + v_col + hd * dim + c]);
  };
  static_assert(DR_TB * DR_COLS <= NT, "a thread stages at most one value of v");
  fetch(0);
  for (int t0 = 0; t0 < count; t0 += DR_TB) {
    const int nt = count - t0 < DR_TB ? count - t0 : DR_TB;
    __syncthreads();                                  // the tokens before are read to their end
#pragma unroll
    for (int x = 0; x < PER; ++x) {
      const int idx = tid + x * NT, t = idx / P, n = idx - t * P;
      if (t < DR_TB) {
        const float u = fk[x] * fi[x];
        s_w[t][n] = fw[x];
        s_au[t][n] = fa[x] * u;
        s_u[t][n] = u;
        s_k[t][n] = fk[x];
        s_r[t][n] = fr[x];
      }
    }
    if (tid < DR_TB * DR_COLS) s_v[tid / DR_COLS][tid % DR_COLS] = fv;
    __syncthreads();
    if (t0 + DR_TB < count) fetch(t0 + DR_TB);
    float mine = 0.f;                                 // lane q keeps token q's result of the column
#pragma unroll
    for (int t = 0; t < DR_TB; ++t) {
      if (t >= nt) break;
      float u[J][VEC], x[J][VEC];
      float dot = 0.f;
#pragma unroll
      for (int j = 0; j < J; ++j) {
        dr_read<VEC>(&s_u[t][16 * VEC * j + VEC * q], u[j]);
#pragma unroll
        for (int e = 0; e < VEC; ++e) dot = __builtin_fmaf(u[j][e], S[j][e], dot);
      }
      dot = dr_sum16(dot);                            // u^T S of this column
      const float v = s_v[t][grp];
#pragma unroll
      for (int j = 0; j < J; ++j) {
        float au[VEC], k[VEC];
        dr_read<VEC>(&s_w[t][16 * VEC * j + VEC * q], x[j]);
        dr_read<VEC>(&s_au[t][16 * VEC * j + VEC * q], au);
        dr_read<VEC>(&s_k[t][16 * VEC * j + VEC * q], k);
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
          const float add = __builtin_fmaf(k[e], v, -(au[e] * dot));
          S[j][e] = __builtin_fmaf(x[j][e], S[j][e], add);
        }
      }
      float o = 0.f;
#pragma unroll
      for (int j = 0; j < J; ++j) {
        dr_read<VEC>(&s_r[t][16 * VEC * j + VEC * q], x[j]);
#pragma unroll
        for (int e = 0; e < VEC; ++e) o = __builtin_fmaf(x[j][e], S[j][e], o);
      }
      o = dr_sum16(o);
      mine = q == t ? o : mine;
    }
    if (col_ok && q < nt) out[((size_t)(first + t0 + q) * nh + hd) * dim + col] = mine;
  }
#pragma unroll
  for (int j = 0; j < J; ++j)
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      const int n = 16 * VEC * j + VEC * q + e;
      if (col_ok && n < dim) st[n] = S[j][e];
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
#define IA_DR(T, V, JJ)                                                                                                  \
  delta_scan_kernel<T, V, JJ><<<grid, 64 * DR_WAVES, 0, stream>>>((const T*)proj, proj_stride, r_col, k_col, v_col, w, a, \
                                                                  inv, state, state_stride, out, seq_starts,             \
                                                                  state_slots, nh, dim)
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
