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
//   ia_delta_chunked     the same for portions of prompts in chunks of DC_T tokens as matrix products (below).
//
// Token after token: a column of S needs nothing of the other columns, so a wave takes four columns: sixteen lanes share a column's
// channels (in registers, a lane dim / 16 of them), the sums over the channels are four rotations within the sixteen
// lanes (every lane ends with the same bits), and a token costs no barrier and no trip through LDS but the reads of
// the token's vectors, which DR_WAVES waves of a workgroup bring into LDS together, DR_TB tokens at a time, the next
// ones' loads in flight meanwhile.  The chain of operations of a column is the same however the tokens are cut into
// steps and whatever else the step holds.
//
// A head's state is kept column by column: slot[head][column][channel].
//
// In chunks: with W_t the product of a chunk's decays up to its token t, S_t = diag(W_t) Z_t turns the recurrence into
//     Z_t = Z_(t-1) - b_t (c_t^T Z_(t-1)) + d_t v_t^T,      b_t = a_t u_t / W_t,  c_t = u_t W_(t-1),  d_t = k_t / W_t,
// so that with S_0 the state before the chunk and the 16 x 16 matrices A = (c_t . b_s), B = (c_t . d_s) below the diagonal
// and F = (e_t . b_s), G = (e_t . d_s) up to it, e_t = r_t W_t, everything the chunk's tokens take from each other is known
// without the state:
//     p = C S_0 + B' V,   C = (I + A)^-1 c,  B' = (I + A)^-1 B;      o = E S_0 + D V,   E = e - F C,  D = G - F B';
//     S_end = diag(W_T) S_0 - (b W_T)^T p + (d W_T)^T V.
// One kernel makes C, E, B', D, -b W_T, d W_T and W_T of every chunk and head side by side; a second walks a request's
// chunks, sixteen columns of a head a workgroup, its waves a tile of sixteen channels (or two) each, on the matrix cores in
// fp32 (v_mfma_f32_16x16x4_f32).  A tile of the state stays in the accumulators: an accumulator's register r of lane
// (q, j) is the state's channel 4 q + r, column j, which is what the second operand wants at a step whose four channels are
// r, 4 + r, 8 + r, 12 + r, and the first operand's records are laid out so that a lane's values of the four steps are 16
// bytes.  The chunks' decays stay above exp(-DC_T decay_scale), so that 1 / W is harmless.  All of it fp32.
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

// ------------------------------------------------------------------------------------------ in chunks
#define DC_T 16          // tokens of a chunk
#define DC_TILE 64       // rows of a tile of the host's list: four chunks
#define DC_MAX_WAVES 8

typedef float dc_f32x4 __attribute__((ext_vector_type(4)));

// A record (one chunk of one head), in floats; `tiles` tiles of 16 channels: C and E [tile][token][16 channels], -b W_T and
// d W_T [tile][channel][16 tokens], W_T [tile][16], B' and D [token][16 tokens].
__host__ __device__ inline long dc_record_floats(int tiles) { return (long)tiles * (4 * 256 + 16) + 2 * 256; }

// The first chunk's record of request s: chunks are counted in the order of the requests from first_request on, four to
// every 64 rows begun.
__device__ __forceinline__ int dc_first_chunk(const int* __restrict__ seq_starts, int first_request, int s) {
  int tiles = 0;
  for (int r = first_request; r < s; ++r) tiles += (seq_starts[r + 1] - seq_starts[r] + DC_TILE - 1) / DC_TILE;
  return tiles * (DC_TILE / DC_T);
}

// grid (tiles x 4, heads), blockDim a multiple of 64: a thread a channel.
template <typename T>
__global__ __launch_bounds__(256, 3) void delta_chunk_prepare_kernel(
    const T* __restrict__ proj, int proj_stride, int r_col, int k_col, const float* __restrict__ w, const float* __restrict__ a,
    const float* __restrict__ inv, const int* __restrict__ seq_starts, const int* __restrict__ tiles_list, int first_request,
    float* __restrict__ records, int nh, int dim) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int tiles = (dim + 15) / 16, DP = tiles * 16, LS = DP + 4;      // LS: a row in LDS
  float* s_c = lds;
  float* s_b = s_c + DC_T * LS;
  float* s_d = s_b + DC_T * LS;
  float* s_e = s_d + DC_T * LS;
  float (*s_m)[16][16] = reinterpret_cast<float (*)[16][16]>(s_e + DC_T * LS);      // A, B, F, G
  const int sub = blockIdx.x & 3, tile = blockIdx.x >> 2, hd = blockIdx.y;
  const int s = tiles_list[2 * tile], row0 = tiles_list[2 * tile + 1] + sub * DC_T;
  const int first = seq_starts[s], qlen = seq_starts[s + 1] - first;
  if (row0 >= qlen) return;
  const int count = qlen - row0 < DC_T ? qlen - row0 : DC_T;
  const int chunk = dc_first_chunk(seq_starts, first_request, s) + row0 / DC_T;
  float* rec = records + ((size_t)chunk * nh + hd) * dc_record_floats(tiles);
  float* rec_c = rec;
  float* rec_e = rec_c + tiles * 256;
  float* rec_b = rec_e + tiles * 256;
  float* rec_d = rec_b + tiles * 256;
  float* rec_w = rec_d + tiles * 256;
  float* rec_bp = rec_w + tiles * 16;
  float* rec_dp = rec_bp + 256;
  const int tid = threadIdx.x, nt = blockDim.x;
  for (int n = tid; n < DP; n += nt) {
    const bool real = n < dim;
    const int nc = real ? n : 0;
    float fw[DC_T], fa[DC_T], fi[DC_T];
    T fk[DC_T], fr[DC_T];
#pragma unroll
    for (int t = 0; t < DC_T; ++t) {                  // rows past the end stand in for none: their values are not used
      const size_t row = (size_t)(first + row0 + (t < count ? t : count - 1)), at = (row * nh + hd) * dim + nc;
      fw[t] = w[at];
      fa[t] = a[at];
      fk[t] = proj[row * proj_stride + k_col + hd * dim + nc];
      fr[t] = proj[row * proj_stride + r_col + hd * dim + nc];
      fi[t] = inv[row * nh + hd];
    }
    float W = 1.f, b[DC_T], d[DC_T];
#pragma unroll
    for (int t = 0; t < DC_T; ++t) {
      const bool ok = real && t < count;
      const float k = ok ? to_float(fk[t]) : 0.f, u = k * fi[t];
      s_c[t * LS + n] = ok ? u * W : 0.f;
      W = ok ? W * fw[t] : W;
      const float iw = 1.0f / W;
      b[t] = ok ? fa[t] * u * iw : 0.f;
      d[t] = k * iw;
      s_b[t * LS + n] = b[t];
      s_d[t * LS + n] = d[t];
      s_e[t * LS + n] = ok ? to_float(fr[t]) * W : 0.f;
    }
    float* ob = rec_b + n * 16;                       // [tile][channel][token]: a channel's sixteen tokens side by side
    float* od = rec_d + n * 16;
#pragma unroll
    for (int t = 0; t < DC_T; t += 4) {
      *reinterpret_cast<float4*>(ob + t) = make_float4(-b[t] * W, -b[t + 1] * W, -b[t + 2] * W, -b[t + 3] * W);
      *reinterpret_cast<float4*>(od + t) = make_float4(d[t] * W, d[t + 1] * W, d[t + 2] * W, d[t + 3] * W);
    }
    rec_w[n] = real ? W : 0.f;
  }
  __syncthreads();
  // ---- A, B, F, G: rows of c or e against rows of b or d
  const int lane = tid & 63, i = lane & 15, q = lane >> 4;
  for (int m = tid >> 6; m < 4; m += nt >> 6) {
    const float* x = (m < 2 ? s_c : s_e) + i * LS + 4 * q;
    const float* y = ((m & 1) ? s_d : s_b) + i * LS + 4 * q;
    dc_f32x4 acc = (dc_f32x4){0.f, 0.f, 0.f, 0.f};
    for (int t = 0; t < tiles; ++t) {
      const float4 xv = *reinterpret_cast<const float4*>(x + 16 * t), yv = *reinterpret_cast<const float4*>(y + 16 * t);
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(xv.x, yv.x, acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(xv.y, yv.y, acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(xv.z, yv.z, acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(xv.w, yv.w, acc, 0, 0, 0);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) s_m[m][4 * q + r][i] = (i < 4 * q + r || (m >= 2 && i == 4 * q + r)) ? acc[r] : 0.f;
  }
  __syncthreads();
  // ---- a thread a column of [c | B] and of [e | G]: forward substitution, then the product with F
  for (int n = tid; n < DP + 16; n += nt) {
    const bool ch = n < DP;
    float y[DC_T];
#pragma unroll
    for (int t = 0; t < DC_T; ++t) {
      float v = ch ? s_c[t * LS + n] : s_m[1][t][n - DP];
#pragma unroll
      for (int x = 0; x < t; ++x) v = __builtin_fmaf(-s_m[0][t][x], y[x], v);
      y[t] = v;
    }
    float* o1 = ch ? rec_c + (n >> 4) * 256 + (n & 15) : rec_bp + (n - DP);       // [tile][token][channel]; [token][token]
    float* o2 = ch ? rec_e + (n >> 4) * 256 + (n & 15) : rec_dp + (n - DP);
#pragma unroll
    for (int t = 0; t < DC_T; ++t) {
      float v = ch ? s_e[t * LS + n] : s_m[3][t][n - DP];
#pragma unroll
      for (int x = 0; x <= t; ++x) v = __builtin_fmaf(-s_m[2][t][x], y[x], v);
      o1[t * 16] = y[t];
      o2[t * 16] = v;
    }
  }
}

// What a wave needs of one chunk.
template <typename T, int TPW>
struct DcOps {
  dc_f32x4 c[TPW], e[TPW], b[TPW], d[TPW], w[TPW], bp, dp;
  T v[4];
};

// grid (heads, requests, slices of 16 columns), blockDim 64 x waves; wave x takes the tiles of channels x TPW ...
template <typename T, int TPW>
__global__ __launch_bounds__(64 * DC_MAX_WAVES) void delta_chunk_scan_kernel(
    const T* __restrict__ proj, int proj_stride, int v_col, float* __restrict__ state, long state_stride,
    float* __restrict__ out, const int* __restrict__ seq_starts, const int* __restrict__ state_slots, int first_request,
    const float* __restrict__ records, int nh, int dim) {
  __shared__ dc_f32x4 part[2][2][DC_MAX_WAVES][64];
  const int hd = blockIdx.x, s = first_request + blockIdx.y, c0 = blockIdx.z * 16;
  const int first = seq_starts[s], count = seq_starts[s + 1] - first;
  if (count <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, nw = blockDim.x >> 6, j = lane & 15, q = lane >> 4;
  const int tiles = (dim + 15) / 16, col = c0 + j;
  const bool col_ok = col < dim;
  const size_t rec_floats = (size_t)dc_record_floats(tiles);
  const float* rec0 = records + ((size_t)dc_first_chunk(seq_starts, first_request, s) * nh + hd) * rec_floats;
  float* st = state + (size_t)state_slots[s] * state_stride + ((size_t)hd * dim + (col_ok ? col : 0)) * dim;
  const bool fours = (dim & 3) == 0;
  int tile[TPW];
  dc_f32x4 S[TPW];
#pragma unroll
  for (int x = 0; x < TPW; ++x) {
    tile[x] = wave * TPW + x;
    S[x] = (dc_f32x4){0.f, 0.f, 0.f, 0.f};
    const int n = tile[x] * 16 + 4 * q;
    if (fours) {
      if (col_ok && n < dim) S[x] = *reinterpret_cast<const dc_f32x4*>(st + n);
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (col_ok && n + r < dim) S[x][r] = st[n + r];
    }
  }
  const int chunks = (count + DC_T - 1) / DC_T;
  const T* vp = proj + v_col + hd * dim + (col_ok ? col : 0);
  auto load = [&](int c, DcOps<T, TPW>& O) {
    const float* rec = rec0 + (size_t)c * nh * rec_floats;
    const int at = j * 16 + 4 * q;
#pragma unroll
    for (int x = 0; x < TPW; ++x) {
      const int t = tile[x] < tiles ? tile[x] : tiles - 1;            // a tile past the head's last: its state stays zero
      O.c[x] = *reinterpret_cast<const dc_f32x4*>(rec + (size_t)t * 256 + at);
      O.e[x] = *reinterpret_cast<const dc_f32x4*>(rec + (size_t)(tiles + t) * 256 + at);
      O.b[x] = *reinterpret_cast<const dc_f32x4*>(rec + (size_t)(2 * tiles + t) * 256 + at);
      O.d[x] = *reinterpret_cast<const dc_f32x4*>(rec + (size_t)(3 * tiles + t) * 256 + at);
      O.w[x] = *reinterpret_cast<const dc_f32x4*>(rec + (size_t)4 * tiles * 256 + t * 16 + 4 * q);
    }
    const float* sq = rec + (size_t)tiles * (4 * 256 + 16);
    O.bp = *reinterpret_cast<const dc_f32x4*>(sq + at);
    O.dp = *reinterpret_cast<const dc_f32x4*>(sq + 256 + at);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = c * DC_T + 4 * q + r;                             // rows past the end meet zeros in every operand
      O.v[r] = vp[(size_t)(first + (t < count ? t : count - 1)) * proj_stride];
    }
  };
  auto work = [&](int c, const DcOps<T, TPW>& O, int buf) {
    float v[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] = to_float(O.v[r]);
    dc_f32x4 P = (dc_f32x4){0.f, 0.f, 0.f, 0.f}, Y = (dc_f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int x = 0; x < TPW; ++x)
      if (tile[x] < tiles) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          P = __builtin_amdgcn_mfma_f32_16x16x4f32(O.c[x][r], S[x][r], P, 0, 0, 0);
          Y = __builtin_amdgcn_mfma_f32_16x16x4f32(O.e[x][r], S[x][r], Y, 0, 0, 0);
        }
      }
    if (wave == 0) {
#pragma unroll
      for (int r = 0; r < 4; ++r) P = __builtin_amdgcn_mfma_f32_16x16x4f32(O.bp[r], v[r], P, 0, 0, 0);
    }
    if (wave == nw - 1) {
#pragma unroll
      for (int r = 0; r < 4; ++r) Y = __builtin_amdgcn_mfma_f32_16x16x4f32(O.dp[r], v[r], Y, 0, 0, 0);
    }
    part[buf][0][wave][lane] = P;
    part[buf][1][wave][lane] = Y;
    dr_barrier();                                     // the other buffer's readers are past it: they met at the chunk before
    P = part[buf][0][0][lane];
    for (int x = 1; x < nw; ++x) P += part[buf][0][x][lane];
#pragma unroll
    for (int x = 0; x < TPW; ++x)
      if (tile[x] < tiles) {
        S[x] *= O.w[x];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          S[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(O.b[x][r], P[r], S[x], 0, 0, 0);
          S[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(O.d[x][r], v[r], S[x], 0, 0, 0);
        }
      }
    if (wave == c % nw) {
      Y = part[buf][1][0][lane];
      for (int x = 1; x < nw; ++x) Y += part[buf][1][x][lane];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = c * DC_T + 4 * q + r;
        if (t < count && col_ok) out[((size_t)(first + t) * nh + hd) * dim + col] = Y[r];
      }
    }
  };
  DcOps<T, TPW> A, B;
  load(0, A);
#pragma unroll
  for (int x = 0; x < TPW; ++x) asm volatile("" : "+v"(S[x]));        // the state has come (see delta_scan_kernel)
  for (int c = 0; c < chunks; c += 2) {               // the next chunk's operands come in while this one is worked on
    if (c + 1 < chunks) load(c + 1, B);
    work(c, A, 0);
    if (c + 1 >= chunks) break;
    if (c + 2 < chunks) load(c + 2, A);
    work(c + 1, B, 1);
  }
#pragma unroll
  for (int x = 0; x < TPW; ++x) {
    const int n = tile[x] * 16 + 4 * q;
    if (fours) {
      if (col_ok && n < dim) *reinterpret_cast<dc_f32x4*>(st + n) = S[x];
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (col_ok && n + r < dim) st[n + r] = S[x][r];
    }
  }
}

// Floats of one chunk's records (all heads): what ia_delta_chunked wants of scratch for every chunk, four chunks to every
// tile of the host's list.
extern "C" long ia_delta_chunk_floats(int nh, int dim) { return (long)nh * dc_record_floats((dim + 15) / 16); }

// ia_delta_scan for the `requests` requests from first_request on, whose rows tiles names: tiles[i] = (request, first row of
// a tile of DC_TILE among its rows), every tile of those requests once, in any order.
extern "C" int ia_delta_chunked(const void* proj, int code, int proj_stride, int r_col, int k_col, int v_col, const float* w,
                                const float* a, const float* inv, float* state, long state_stride, float* out,
                                const int* seq_starts, const int* state_slots, const int* tiles, int num_tiles,
                                int first_request, int requests, float* records, int nh, int dim, hipStream_t stream) {
  if (num_tiles == 0 || requests == 0) return IA_OK;
  if (!proj || !w || !a || !inv || !state || !out || !seq_starts || !state_slots || !tiles || !records || num_tiles < 0 ||
      first_request < 0 || requests < 0 || nh <= 0 || dim <= 0 || r_col < 0 || k_col < 0 || v_col < 0 ||
      proj_stride < r_col + nh * dim || proj_stride < k_col + nh * dim || proj_stride < v_col + nh * dim ||
      state_stride < ia_delta_state_floats(nh, dim) || (code != IA_F32 && code != IA_BF16) ||
      (((uintptr_t)records | (uintptr_t)state) & 15) || ((dim & 3) == 0 && (state_stride & 3)))
    return IA_ERR_BAD_ARG;
  if (dim > 256 || requests > 65535 || nh > 65535 || num_tiles > 0x1fffffff) return IA_ERR_UNSUPPORTED;
  const int t16 = (dim + 15) / 16, DP = t16 * 16;
  const int threads = (DP + 63) / 64 * 64;
  const size_t lds = sizeof(float) * (4 * (size_t)DC_T * (DP + 4) + 4 * 256);
  const int tpw = t16 > DC_MAX_WAVES ? 2 : 1, waves = (t16 + tpw - 1) / tpw;
  const dim3 pgrid((unsigned)num_tiles * 4, (unsigned)nh), sgrid((unsigned)nh, (unsigned)requests, (unsigned)t16);
#define IA_DC(T)                                                                                                             \
  do {                                                                                                                       \
    if (lds > 64 * 1024)                                                                                                     \
      (void)hipFuncSetAttribute((const void*)delta_chunk_prepare_kernel<T>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); \
    delta_chunk_prepare_kernel<T><<<pgrid, threads, lds, stream>>>((const T*)proj, proj_stride, r_col, k_col, w, a, inv,      \
                                                                   seq_starts, tiles, first_request, records, nh, dim);      \
    IA_LAUNCH_CHECK();                                                                                                       \
    if (tpw == 1)                                                                                                            \
      delta_chunk_scan_kernel<T, 1><<<sgrid, 64 * waves, 0, stream>>>((const T*)proj, proj_stride, v_col, state, state_stride, \
                                                                      out, seq_starts, state_slots, first_request, records,  \
                                                                      nh, dim);                                              \
    else                                                                                                                     \
      delta_chunk_scan_kernel<T, 2><<<sgrid, 64 * waves, 0, stream>>>((const T*)proj, proj_stride, v_col, state, state_stride, \
                                                                      out, seq_starts, state_slots, first_request, records,  \
                                                                      nh, dim);                                              \
  } while (0)
  if (code == IA_F32) IA_DC(float);
  else IA_DC(bf16_t);
#undef IA_DC
  IA_LAUNCH_CHECK();
  return IA_OK;
}

#include "op_call.h"
IA_OP(ia_delta_tanh_rows)
IA_OP(ia_delta_prepare)
IA_OP(ia_delta_scan)
IA_OP(ia_delta_chunked)
