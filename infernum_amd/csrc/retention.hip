// Retention: a recurrence per head over a state S [dim, vdim] of fp32 values with one fixed decay a head,
//     S_t = g S_(t-1) + k_t v_t^T,      o_t = S_t^T q_t,
// q and k rotated by their position, k times a factor, and what follows it: every head's o divided by its root mean
// square over vdim, times a factor, times silu(gate), rounded once into the activations' type.
//
//   ia_rotation_table    cosine and sine of position * frequency for every token of a step and every pair: made once a
//                        step for all layers and heads that rotate alike;
//   ia_retention_step    the recurrence token after token from the request's state slot, which is left moved on: single
//                        tokens, the 32-bit path, head sizes that the chunks do not take.  A workgroup per (request, head)
//                        passes over the head's state once a token;
//   ia_retention_chunked the same for portions of prompts as matrix products over tiles of RET_TILE rows that run side by
//                        side.  With i, j the rows of a tile of L rows, counted from 0, that starts from the state S0:
//                            o_i = sum_{j <= i} g^(i - j) (q_i . k_j) v_j + g^(i + 1) S0^T q_i,
//                            S   = g^L S0 + sum_j g^(L - 1 - j) k_j v_j^T.
//                        A first kernel leaves what every tile but a request's last adds to the state, a second walks a
//                        request's tiles and leaves each the state before it, a third writes the rows, the norm and the
//                        gate among them, and the last tile's the slot.
//
// Rotated queries and keys, decays, sums and the state are fp32 (the products on v_mfma_f32_16x16x4_f32); the values are
// the activations as the projection left them.  The state lies [head][dim][vdim] in the slot.
#include "common.h"

typedef float rt_f32x4 __attribute__((ext_vector_type(4)));

#define RET_TILE 64       // rows of a tile
#define RET_GS 68         // row stride of a tile's [L, L] matrix in LDS, floats
#define RET_MAX_DIM 256   // head sizes of the chunks
#define RET_GROUPS 4      // groups of four values whose loads a thread asks for together
#define RET_STEP_MAX 1024 // head sizes of the step

__global__ __launch_bounds__(256) void rotation_table_kernel(const int* __restrict__ positions, const void* __restrict__ freq,
                                                             int freq_f64, float2* __restrict__ out, int N, int half) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= N * half) return;
  const int n = i / half;
  float sn, cs;
  rope_sincos(positions[n], freq, freq_f64, i - n * half, sn, cs);
  out[i] = make_float2(cs, sn);
}

// out: [N, half] pairs (cosine, sine), fp32
extern "C" int ia_rotation_table(const int* positions, const void* freq, int freq_f64, float* out, int N, int half,
                                 hipStream_t stream) {
  if (N == 0) return IA_OK;
  if (!positions || !freq || !out || N < 0 || half <= 0 || (long)N * half > 0x7fffffffL) return IA_ERR_BAD_ARG;
  rotation_table_kernel<<<(N * half + 255) / 256, 256, 0, stream>>>(positions, freq, freq_f64, (float2*)out, N, half);
  IA_LAUNCH_CHECK();
  return IA_OK;
}

struct RetArgs {
  const float* table;            // [N, rot / 2, 2], or null with rot 0
  const float* decay;            // [2, nh]: the decays, then their logarithms to the base 2
  float* state;
  long state_stride;
  const int* seq_starts;
  const int* state_slots;
  int proj_stride, q_col, k_col, v_col, g_col, out_stride, nh, dim, vdim, rot;
  float k_factor, eps, o_factor;
};

// g^n for a whole n >= 0 (a decay of zero has the logarithm -infinity)
__device__ __forceinline__ float ret_pow(float log2_decay, int n) { return n == 0 ? 1.0f : exp2f(log2_decay * (float)n); }

// Value i of a head behind the rotation of halves: `row` its dim values, `cs` the token's table.
template <typename T>
__device__ __forceinline__ float ret_rotated(const T* __restrict__ row, const float2* __restrict__ cs, int i, int rot) {
  if (i >= rot) return to_float(row[i]);
  const int half = rot >> 1;
  const bool low = i < half;
  const float2 a = cs[low ? i : i - half];
  const float x = to_float(row[i]), y = to_float(row[low ? i + half : i - half]);
  float lo, hi;
  rope_pair(low ? x : y, low ? y : x, a.x, a.y, lo, hi);
  return low ? lo : hi;
}

// ------------------------------------------------------------------------------------------ token after token
// grid (heads, requests), 256 threads.  V: values of a state row that a thread takes together.
#define RET_ROWS 8        // rows of the state whose loads are in flight together
template <typename T, int V>
__global__ __launch_bounds__(256) void retention_step_kernel(const T* __restrict__ proj, T* __restrict__ out, RetArgs P) {
  extern __shared__ __attribute__((aligned(16))) float ret_lds[];
  __shared__ float s_red[4];
  const int hd = blockIdx.x, s = blockIdx.y, tid = threadIdx.x;
  const int first = P.seq_starts[s], count = P.seq_starts[s + 1] - first;
  if (count <= 0) return;
  const int dim = P.dim, vdim = P.vdim, cols = vdim / V;
  const int lanes = cols < 256 ? cols : 256, parts = 256 / lanes;
  float* qs = ret_lds;                               // [dim]
  float* ks = qs + dim;                              // [dim]
  float* acc_s = ks + dim;                           // [parts][vdim], then [vdim]
  float* S = P.state + (size_t)P.state_slots[s] * P.state_stride + (size_t)hd * dim * vdim;
  const float g = P.decay[hd];
  const int part = tid / lanes, lane = tid - part * lanes;
  for (int t = 0; t < count; ++t) {
    const size_t n = (size_t)(first + t);
    const T* row = proj + n * P.proj_stride;
    const float2* cs = reinterpret_cast<const float2*>(P.table) + n * (P.rot >> 1);
    for (int i = tid; i < dim; i += 256) {
      qs[i] = ret_rotated(row + P.q_col + hd * dim, cs, i, P.rot);
      ks[i] = ret_rotated(row + P.k_col + hd * dim, cs, i, P.rot) * P.k_factor;
    }
    __syncthreads();
    if (part < parts) {
      for (int c = lane; c < cols; c += lanes) {
        float v[V], acc[V];
        const T* vr = row + P.v_col + (size_t)hd * vdim + c * V;
#pragma unroll
        for (int e = 0; e < V; ++e) {
          v[e] = to_float(vr[e]);
          acc[e] = 0.f;
        }
        for (int r0 = part; r0 < dim; r0 += parts * RET_ROWS) {
          float st[RET_ROWS][V];
#pragma unroll
          for (int k = 0; k < RET_ROWS; ++k) {
            const int r = r0 + k * parts;
            const float* p = S + (size_t)(r < dim ? r : r0) * vdim + c * V;
            if (V == 4) {
              const float4 w = *reinterpret_cast<const float4*>(p);
              st[k][0] = w.x; st[k][V > 1 ? 1 : 0] = w.y; st[k][V > 2 ? 2 : 0] = w.z; st[k][V > 3 ? 3 : 0] = w.w;
            } else {
              st[k][0] = p[0];
            }
          }
#pragma unroll
          for (int k = 0; k < RET_ROWS; ++k) {
            const int r = r0 + k * parts;
            if (r < dim) {
              const float kk = ks[r], qq = qs[r];
#pragma unroll
              for (int e = 0; e < V; ++e) {
                st[k][e] = __builtin_fmaf(g, st[k][e], kk * v[e]);
                acc[e] = __builtin_fmaf(st[k][e], qq, acc[e]);
              }
              float* p = S + (size_t)r * vdim + c * V;
              if (V == 4) *reinterpret_cast<float4*>(p) = make_float4(st[k][0], st[k][V > 1 ? 1 : 0], st[k][V > 2 ? 2 : 0], st[k][V > 3 ? 3 : 0]);
              else p[0] = st[k][0];
            }
          }
        }
#pragma unroll
        for (int e = 0; e < V; ++e) acc_s[(size_t)part * vdim + c * V + e] = acc[e];
      }
    }
    __syncthreads();
    float ss = 0.f;
    for (int i = tid; i < vdim; i += 256) {
      float o = acc_s[i];
      for (int k = 1; k < parts; ++k) o += acc_s[(size_t)k * vdim + i];
      acc_s[i] = o;
      ss = __builtin_fmaf(o, o, ss);
    }
    ss = block_sum<256>(ss, s_red);
    const float f = P.o_factor / sqrtf(ss / (float)vdim + P.eps);
    const T* gr = row + P.g_col + (size_t)hd * vdim;
    T* orow = out + n * P.out_stride + (size_t)hd * vdim;
    for (int i = tid; i < vdim; i += 256) {
      const float gate = to_float(gr[i]);
      orow[i] = from_float<T>(acc_s[i] * f * (gate / (1.0f + expf(-gate))));
    }
    __syncthreads();                                   // queries, keys and sums are free for the next token
  }
}

// ------------------------------------------------------------------------------------------ in tiles
__host__ __device__ inline int ret_stride(int d) { return d % 32 == 0 ? d + 16 : d; }       // floats of a row in LDS
__host__ __device__ inline int ret_vstride(int vd) { return vd + 8; }                       // bf16 of a row in LDS

// The record of a tile: the tiles of the requests from ``first_request`` on, in the order of the requests and their rows.
__device__ __forceinline__ int ret_record(const int* __restrict__ seq_starts, int first_request, int s, int r0) {
  int before = 0;
  for (int r = first_request; r < s; ++r) before += (seq_starts[r + 1] - seq_starts[r] + RET_TILE - 1) / RET_TILE;
  return before + r0 / RET_TILE;
}

// Rows first .. first + count - 1 of a head's queries or keys (from column `col`), rotated, times `factor`, into LDS; zeros
// up to RET_TILE rows.  Four values a thread: dim is a multiple of 16, and so that a group's partners are a group, rot / 2
// a multiple of 4 (QUADS), or one value a thread.
template <bool QUADS>
__device__ __forceinline__ void ret_stage(const bf16_t* __restrict__ proj, const RetArgs& P, int col, int first, int count,
                                          float factor, float* __restrict__ dst, int stride, int tid, int threads) {
  const int dim = P.dim, half = P.rot >> 1;
  if (!QUADS) {
    for (int i = tid; i < RET_TILE * dim; i += threads) {
      const int r = i / dim, c = i - r * dim;
      const size_t n = (size_t)(first + r);
      dst[r * stride + c] = r < count ? factor * ret_rotated(proj + n * P.proj_stride + col,
                                                             reinterpret_cast<const float2*>(P.table) + n * half, c, P.rot) : 0.f;
    }
    return;
  }
  // RET_GROUPS groups of four values of a thread, their loads all asked for before the first is used: rows past the last
  // load the last one and are zeroed behind it, values that are not rotated load themselves as their partners
  const int quads = dim / 4, total = RET_TILE * quads;
  for (int i0 = tid; i0 < total; i0 += RET_GROUPS * threads) {
    uint2 w[RET_GROUPS], u[RET_GROUPS];
    float4 ca[RET_GROUPS], cb[RET_GROUPS];
#pragma unroll
    for (int k = 0; k < RET_GROUPS; ++k) {
      const int i = i0 + k * threads < total ? i0 + k * threads : i0;
      const int r = i / quads, c = (i - r * quads) * 4;
      const size_t n = (size_t)(first + (r < count ? r : count - 1));
      const bf16_t* row = proj + n * P.proj_stride + col;
      const bool low = c < half, turned = c < P.rot;
      w[k] = *reinterpret_cast<const uint2*>(row + c);
      u[k] = *reinterpret_cast<const uint2*>(row + (turned ? (low ? c + half : c - half) : c));
      if (turned) {
        const float4* cs = reinterpret_cast<const float4*>(P.table + (n * half + (low ? c : c - half)) * 2);
        ca[k] = cs[0];
        cb[k] = cs[1];
      } else {
        ca[k] = cb[k] = make_float4(1.f, 0.f, 1.f, 0.f);
      }
    }
#pragma unroll
    for (int k = 0; k < RET_GROUPS; ++k) {
      const int i = i0 + k * threads;
      if (i >= total) break;
      const int r = i / quads, c = (i - r * quads) * 4;
      float x[4] = {__uint_as_float(w[k].x << 16), __uint_as_float(w[k].x & 0xffff0000u), __uint_as_float(w[k].y << 16),
                    __uint_as_float(w[k].y & 0xffff0000u)};
      if (c < P.rot) {
        const bool low = c < half;
        const float y[4] = {__uint_as_float(u[k].x << 16), __uint_as_float(u[k].x & 0xffff0000u), __uint_as_float(u[k].y << 16),
                            __uint_as_float(u[k].y & 0xffff0000u)};
        const float cv[4] = {ca[k].x, ca[k].z, cb[k].x, cb[k].z}, sv[4] = {ca[k].y, ca[k].w, cb[k].y, cb[k].w};
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          float lo, hi;
          rope_pair(low ? x[e] : y[e], low ? y[e] : x[e], cv[e], sv[e], lo, hi);
          x[e] = low ? lo : hi;
        }
      }
      const float f = r < count ? factor : 0.f;
      *reinterpret_cast<float4*>(dst + r * stride + c) = make_float4(x[0] * f, x[1] * f, x[2] * f, x[3] * f);
    }
  }
}

__device__ __forceinline__ void ret_stage_values(const bf16_t* __restrict__ proj, const RetArgs& P, int col, int first, int count,
                                                 uint16_t* __restrict__ dst, int stride, int tid, int threads) {
  const int pieces = P.vdim / 8;
  for (int i = tid; i < RET_TILE * pieces; i += threads) {
    const int r = i / pieces, c = (i - r * pieces) * 8;
    uint4 v = make_uint4(0, 0, 0, 0);
    if (r < count) v = *reinterpret_cast<const uint4*>(proj + (size_t)(first + r) * P.proj_stride + col + c);
    *reinterpret_cast<uint4*>(dst + r * stride + c) = v;
  }
}

// What a tile of `count` rows makes of the state: W <- keep R + sum_j g^(count - 1 - j) k_j v_j^T (R null: nothing kept).
// ks [RET_TILE][kst] fp32, vs [RET_TILE][vst] bf16, pw[n] = g^n; eight waves take blocks of 32 x 32 of the state in turn.
__device__ __forceinline__ void ret_state(const float* __restrict__ ks, int kst, const uint16_t* __restrict__ vs, int vst,
                                          const float* __restrict__ pw, int count, float keep, const float* __restrict__ R,
                                          float* __restrict__ W, int dim, int vdim, int wave, int lane) {
  const int l15 = lane & 15, kk = lane >> 4;
  const int nb = (dim + 31) / 32, cb = (vdim + 31) / 32;
  for (int b = wave; b < nb * cb; b += 8) {
    const int n0 = (b / cb) * 32, c0 = (b - (b / cb) * cb) * 32;
    const bool n2 = n0 + 16 < dim, c2 = c0 + 16 < vdim;
    const int n1 = n2 ? n0 + 16 : n0, c1 = c2 ? c0 + 16 : c0;
    rt_f32x4 a00 = {0.f, 0.f, 0.f, 0.f}, a01 = a00, a10 = a00, a11 = a00;
#pragma unroll 4
    for (int j0 = 0; j0 < RET_TILE; j0 += 4) {
      const int j = j0 + kk;
      const float w = j < count ? pw[count - 1 - j] : 0.f;
      const float k0 = ks[j * kst + n0 + l15] * w, k1 = ks[j * kst + n1 + l15] * w;
      const float v0 = __uint_as_float((uint32_t)vs[j * vst + c0 + l15] << 16), v1 = __uint_as_float((uint32_t)vs[j * vst + c1 + l15] << 16);
      a00 = __builtin_amdgcn_mfma_f32_16x16x4f32(k0, v0, a00, 0, 0, 0);
      a01 = __builtin_amdgcn_mfma_f32_16x16x4f32(k0, v1, a01, 0, 0, 0);
      a10 = __builtin_amdgcn_mfma_f32_16x16x4f32(k1, v0, a10, 0, 0, 0);
      a11 = __builtin_amdgcn_mfma_f32_16x16x4f32(k1, v1, a11, 0, 0, 0);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const size_t p0 = (size_t)(n0 + 4 * kk + r) * vdim + l15, p1 = (size_t)(n1 + 4 * kk + r) * vdim + l15;
      W[p0 + c0] = R ? __builtin_fmaf(keep, R[p0 + c0], a00[r]) : a00[r];
      if (c2) W[p0 + c1] = R ? __builtin_fmaf(keep, R[p0 + c1], a01[r]) : a01[r];
      if (n2) {
        W[p1 + c0] = R ? __builtin_fmaf(keep, R[p1 + c0], a10[r]) : a10[r];
        if (c2) W[p1 + c1] = R ? __builtin_fmaf(keep, R[p1 + c1], a11[r]) : a11[r];
      }
    }
  }
}

// grid (heads, tiles), 512 threads
template <bool QUADS>
__global__ __launch_bounds__(512) void retention_adds_kernel(const bf16_t* __restrict__ proj, const int* __restrict__ tiles,
                                                             int first_request, float* __restrict__ records, long record_stride,
                                                             RetArgs P) {
  extern __shared__ __attribute__((aligned(16))) float ret_lds[];
  __shared__ float pw[RET_TILE];
  const int hd = blockIdx.x, s = tiles[2 * blockIdx.y], r0 = tiles[2 * blockIdx.y + 1], tid = threadIdx.x;
  const int count = P.seq_starts[s + 1] - P.seq_starts[s];
  if (r0 + RET_TILE >= count) return;                  // a request's last tile adds nothing that anyone reads
  const int first = P.seq_starts[s] + r0, kst = ret_stride(P.dim), vst = ret_vstride(P.vdim);
  float* ks = ret_lds;
  uint16_t* vs = reinterpret_cast<uint16_t*>(ks + RET_TILE * kst);
  if (tid < RET_TILE) pw[tid] = ret_pow(P.decay[P.nh + hd], tid);
  ret_stage<QUADS>(proj, P, P.k_col + hd * P.dim, first, RET_TILE, P.k_factor, ks, kst, tid, 512);
  ret_stage_values(proj, P, P.v_col + hd * P.vdim, first, RET_TILE, vs, vst, tid, 512);
  __syncthreads();
  float* W = records + (size_t)ret_record(P.seq_starts, first_request, s, r0) * record_stride + (size_t)hd * P.dim * P.vdim;
  ret_state(ks, kst, vs, vst, pw, RET_TILE, 0.f, nullptr, W, P.dim, P.vdim, tid >> 6, tid & 63);
}

// grid (blocks of 256 of the heads' values, tiles), 256 threads: the workgroups of a request's first tile walk its tiles.
#define RET_AHEAD 8
__global__ __launch_bounds__(256) void retention_chain_kernel(const int* __restrict__ tiles, int first_request,
                                                              float* __restrict__ records, long record_stride, RetArgs P) {
  if (tiles[2 * blockIdx.y + 1] != 0) return;
  const int s = tiles[2 * blockIdx.y], rows = P.seq_starts[s + 1] - P.seq_starts[s];
  const int e = blockIdx.x * 256 + threadIdx.x, per = P.dim * P.vdim;
  if (e >= P.nh * per) return;
  const float keep = ret_pow(P.decay[P.nh + e / per], RET_TILE);
  const int count = (rows + RET_TILE - 1) / RET_TILE;
  float S = P.state[(size_t)P.state_slots[s] * P.state_stride + e];
  float* R = records + (size_t)ret_record(P.seq_starts, first_request, s, 0) * record_stride + e;
  for (int j0 = 0; j0 < count; j0 += RET_AHEAD) {
    float U[RET_AHEAD];
#pragma unroll
    for (int k = 0; k < RET_AHEAD; ++k) U[k] = j0 + k < count - 1 ? R[(size_t)(j0 + k) * record_stride] : 0.f;
#pragma unroll
    for (int k = 0; k < RET_AHEAD; ++k) {
      if (j0 + k >= count) break;
      R[(size_t)(j0 + k) * record_stride] = S;
      S = __builtin_fmaf(keep, S, U[k]);
    }
  }
}

// The rows of the tile for column tiles of 16 values: a wave takes RT of the four row tiles of one column tile (a job).
template <int RT>
__device__ __forceinline__ void ret_rows(const float* __restrict__ qs, int kst, const float* __restrict__ G,
                                         const uint16_t* __restrict__ vs, int vst, const float* __restrict__ pw,
                                         const float* __restrict__ S, int dim, int vdim, int ct, int rt0, int lane,
                                         rt_f32x4 (&acc)[4]) {
  const int l15 = lane & 15, kk = lane >> 4;
  const float* sp = S + (size_t)(4 * kk) * vdim + 16 * ct + l15;
#pragma unroll
  for (int a = 0; a < RT; ++a) acc[a] = (rt_f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int n0 = 0; n0 < dim; n0 += 16) {
    float b[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) b[r] = sp[(size_t)(n0 + r) * vdim];
#pragma unroll
    for (int a = 0; a < RT; ++a) {
      const rt_f32x4 q = *reinterpret_cast<const rt_f32x4*>(qs + (16 * (rt0 + a) + l15) * kst + n0 + 4 * kk);
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[a] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[r], b[r], acc[a], 0, 0, 0);
    }
  }
#pragma unroll
  for (int a = 0; a < RT; ++a)
#pragma unroll
    for (int r = 0; r < 4; ++r) acc[a][r] *= pw[16 * (rt0 + a) + 4 * kk + r + 1];
  for (int jt = 0; jt < rt0 + RT; ++jt) {
    float b[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) b[r] = __uint_as_float((uint32_t)vs[(16 * jt + 4 * kk + r) * vst + 16 * ct + l15] << 16);
#pragma unroll
    for (int a = 0; a < RT; ++a) {
      if (jt > rt0 + a) continue;
      const rt_f32x4 q = *reinterpret_cast<const rt_f32x4*>(G + (16 * (rt0 + a) + l15) * RET_GS + 16 * jt + 4 * kk);
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[a] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[r], b[r], acc[a], 0, 0, 0);
    }
  }
}

// grid (heads, tiles), 512 threads.  RT: row tiles of a job (4, 2 or 1, so that eight waves have jobs); JOBS: jobs of a wave.
template <bool QUADS, int RT, int JOBS>
__global__ __launch_bounds__(512) void retention_rows_kernel(const bf16_t* __restrict__ proj, bf16_t* __restrict__ out,
                                                             const int* __restrict__ tiles, int first_request,
                                                             const float* __restrict__ records, long record_stride, RetArgs P) {
  extern __shared__ __attribute__((aligned(16))) float ret_lds[];
  __shared__ float pw[RET_TILE + 1], stat[RET_TILE][RET_MAX_DIM / 16 + 1], inv[RET_TILE];
  const int hd = blockIdx.x, s = tiles[2 * blockIdx.y], r0 = tiles[2 * blockIdx.y + 1], tid = threadIdx.x;
  const int rows = P.seq_starts[s + 1] - P.seq_starts[s], left = rows - r0;
  const bool last = left <= RET_TILE;
  const int count = last ? left : RET_TILE, first = P.seq_starts[s] + r0;
  if (count <= 0) return;
  const int dim = P.dim, vdim = P.vdim, kst = ret_stride(dim), vst = ret_vstride(vdim);
  const int wave = tid >> 6, lane = tid & 63, l15 = lane & 15, kk = lane >> 4;
  float* qs = ret_lds;                                              // [TILE][kst]
  float* ks = qs + RET_TILE * kst;                                  // [TILE][kst]
  float* G = ks + RET_TILE * kst;                                   // [TILE][GS]
  uint16_t* vs = reinterpret_cast<uint16_t*>(G + RET_TILE * RET_GS);// [TILE][vst]
  if (tid <= RET_TILE) pw[tid] = ret_pow(P.decay[P.nh + hd], tid);
  ret_stage<QUADS>(proj, P, P.q_col + hd * dim, first, count, 1.0f, qs, kst, tid, 512);
  ret_stage<QUADS>(proj, P, P.k_col + hd * dim, first, count, P.k_factor, ks, kst, tid, 512);
  ret_stage_values(proj, P, P.v_col + hd * vdim, first, count, vs, vst, tid, 512);
  __syncthreads();
  // ---- G[i][j] = g^(i - j) (q_i . k_j) for j <= i: the ten tiles of 16 x 16 on and under the diagonal over eight waves
  for (int t = wave; t < 10; t += 8) {
    const int it = t < 1 ? 0 : t < 3 ? 1 : t < 6 ? 2 : 3, jt = t - (it * (it + 1) >> 1);
    rt_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    const float* qp = qs + (16 * it + l15) * kst + 4 * kk;
    const float* kp = ks + (16 * jt + l15) * kst + 4 * kk;
#pragma unroll 2
    for (int n0 = 0; n0 < dim; n0 += 16) {
      const rt_f32x4 a = *reinterpret_cast<const rt_f32x4*>(qp + n0), b = *reinterpret_cast<const rt_f32x4*>(kp + n0);
#pragma unroll
      for (int r = 0; r < 4; ++r) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[r], b[r], acc, 0, 0, 0);
    }
    const int j = 16 * jt + l15;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * it + 4 * kk + r;
      G[i * RET_GS + j] = j <= i ? acc[r] * pw[i - j] : 0.f;
    }
  }
  __syncthreads();
  const float* S = records + (size_t)ret_record(P.seq_starts, first_request, s, r0) * record_stride + (size_t)hd * dim * vdim;
  constexpr int SPLIT = 4 / RT;
  const int ctiles = vdim / 16, jobs = ctiles * SPLIT;
  rt_f32x4 acc[JOBS][4];
  bf16_t gates[JOBS][RT][4];                            // asked for before the products, needed behind them
#pragma unroll
  for (int b = 0; b < JOBS; ++b) {
    const int job = wave + 8 * b;
    if (job >= jobs) break;
    const int ct = job / SPLIT, rt0 = (job - ct * SPLIT) * RT;
#pragma unroll
    for (int a = 0; a < RT; ++a)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * (rt0 + a) + 4 * kk + r;
        gates[b][a][r] = proj[(size_t)(first + (i < count ? i : count - 1)) * P.proj_stride + P.g_col + hd * vdim + 16 * ct + l15];
      }
    ret_rows<RT>(qs, kst, G, vs, vst, pw, S, dim, vdim, ct, rt0, lane, acc[b]);
#pragma unroll
    for (int a = 0; a < RT; ++a)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float q = acc[b][a][r] * acc[b][a][r];
#pragma unroll
        for (int o = 1; o < 16; o <<= 1) q += __shfl_xor(q, o, IA_WAVE);
        if (l15 == 0) stat[16 * (rt0 + a) + 4 * kk + r][ct] = q;
      }
  }
  __syncthreads();
  if (tid < RET_TILE) {
    float q = stat[tid][0];
    for (int c = 1; c < ctiles; ++c) q += stat[tid][c];
    inv[tid] = P.o_factor / sqrtf(q / (float)vdim + P.eps);
  }
  __syncthreads();
#pragma unroll
  for (int b = 0; b < JOBS; ++b) {
    const int job = wave + 8 * b;
    if (job >= jobs) break;
    const int ct = job / SPLIT, rt0 = (job - ct * SPLIT) * RT;
#pragma unroll
    for (int a = 0; a < RT; ++a)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * (rt0 + a) + 4 * kk + r;
        if (i >= count) continue;
        const size_t n = (size_t)(first + i);
        const int c = hd * vdim + 16 * ct + l15;
        const float gate = to_float(gates[b][a][r]);
        const float silu = gate * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * gate));
        out[n * P.out_stride + c] = from_float<bf16_t>(acc[b][a][r] * inv[i] * silu);
      }
  }
  if (last) {
    float* W = P.state + (size_t)P.state_slots[s] * P.state_stride + (size_t)hd * dim * vdim;
    ret_state(ks, kst, vs, vst, pw, count, pw[count], S, W, dim, vdim, wave, lane);
  }
}

// ------------------------------------------------------------------------------------------ C interface
// Floats a request's slot holds for one layer run.
extern "C" long ia_retention_state_floats(int nh, int dim, int vdim) { return (long)nh * dim * vdim; }

static bool ret_bad(const RetArgs& P) {
  return !P.decay || !P.state || !P.seq_starts || !P.state_slots || P.nh <= 0 || P.dim <= 0 || P.vdim <= 0 || P.rot < 0 ||
         P.rot > P.dim || (P.rot & 1) || (P.rot > 0 && !P.table) || P.q_col < 0 || P.k_col < 0 || P.v_col < 0 || P.g_col < 0 ||
         P.proj_stride < P.q_col + P.nh * P.dim || P.proj_stride < P.k_col + P.nh * P.dim ||
         P.proj_stride < P.v_col + P.nh * P.vdim || P.proj_stride < P.g_col + P.nh * P.vdim || P.out_stride < P.nh * P.vdim ||
         P.state_stride < ia_retention_state_floats(P.nh, P.dim, P.vdim) || !(P.eps > 0.f);
}

// proj: rows of proj_stride values (code: their type) holding q and k (nh dim values each from q_col, k_col), v and the
// gates (nh vdim each from v_col, g_col); table: ia_rotation_table for rot / 2 pairs; decay fp32 [2, nh]: the decays
// and their logarithms to the base 2; out: rows of
// out_stride values.  Requests 0 .. B - 1.
extern "C" int ia_retention_step(const void* proj, int code, int proj_stride, int q_col, int k_col, int v_col, int g_col,
                                 const float* table, int rot, float k_factor, const float* decay, float eps,
                                 float o_factor, float* state, long state_stride, void* out, int out_stride,
                                 const int* seq_starts, const int* state_slots, int B, int nh, int dim, int vdim,
                                 hipStream_t stream) {
  if (B == 0) return IA_OK;
  const RetArgs P{table, decay, state, state_stride, seq_starts, state_slots, proj_stride, q_col, k_col, v_col, g_col,
                  out_stride, nh, dim, vdim, rot, k_factor, eps, o_factor};
  if (B < 0 || !proj || !out || ret_bad(P)) return IA_ERR_BAD_ARG;
  if (B > 65535 || dim > RET_STEP_MAX || vdim > RET_STEP_MAX) return IA_ERR_UNSUPPORTED;
  const bool vec = vdim % 4 == 0 && state_stride % 4 == 0 && !((uintptr_t)state & 15);
  const int cols = vec ? vdim / 4 : vdim, lanes = cols < 256 ? cols : 256;
  const size_t lds = sizeof(float) * (2 * (size_t)dim + (size_t)(256 / lanes) * vdim);
  if (lds > 64 * 1024) return IA_ERR_UNSUPPORTED;
  const dim3 grid((unsigned)nh, (unsigned)B);
#define IA_RS(T, V) retention_step_kernel<T, V><<<grid, 256, lds, stream>>>((const T*)proj, (T*)out, P)
  if (code == IA_F32) {
    if (vec) IA_RS(float, 4);
    else IA_RS(float, 1);
  } else if (code == IA_BF16) {
    if (vec) IA_RS(bf16_t, 4);
    else IA_RS(bf16_t, 1);
  } else
    return IA_ERR_BAD_ARG;
#undef IA_RS
  IA_LAUNCH_CHECK();
  return IA_OK;
}

static size_t ret_rows_lds(int dim, int vdim) {
  return sizeof(float) * ((size_t)2 * RET_TILE * ret_stride(dim) + RET_TILE * RET_GS) + 2 * (size_t)RET_TILE * ret_vstride(vdim);
}

// Whether ia_retention_chunked takes these sizes (otherwise ia_retention_step does the portions too).
extern "C" int ia_retention_chunked_takes(int nh, int dim, int vdim, int proj_stride, int q_col, int k_col, int v_col) {
  return nh > 0 && dim % 16 == 0 && vdim % 16 == 0 && dim >= 16 && vdim >= 16 && dim <= RET_MAX_DIM && vdim <= RET_MAX_DIM &&
         proj_stride % 8 == 0 && q_col % 8 == 0 && k_col % 8 == 0 && v_col % 8 == 0 && ret_rows_lds(dim, vdim) <= 150 * 1024;
}

// The requests that the tiles name: tiles[i] = (request, first row of a tile of RET_TILE among the request's rows) in any
// order, every tile of the requests first_request .. once.  records: fp32 [num_tiles, record_stride].
extern "C" int ia_retention_chunked(const void* proj, int code, int proj_stride, int q_col, int k_col, int v_col, int g_col,
                                    const float* table, int rot, float k_factor, const float* decay, float eps,
                                    float o_factor, float* state, long state_stride, void* out, int out_stride,
                                    const int* seq_starts, const int* state_slots, const int* tiles, int num_tiles,
                                    int first_request, float* records, long record_stride, int nh, int dim, int vdim,
                                    hipStream_t stream) {
  if (num_tiles == 0) return IA_OK;
  const RetArgs P{table, decay, state, state_stride, seq_starts, state_slots, proj_stride, q_col, k_col, v_col, g_col,
                  out_stride, nh, dim, vdim, rot, k_factor, eps, o_factor};
  if (num_tiles < 0 || first_request < 0 || !proj || !out || !tiles || !records || ret_bad(P) ||
      record_stride < ia_retention_state_floats(nh, dim, vdim))
    return IA_ERR_BAD_ARG;
  if (code != IA_BF16 || num_tiles > 65535 || ((uintptr_t)proj & 15) ||
      !ia_retention_chunked_takes(nh, dim, vdim, proj_stride, q_col, k_col, v_col))
    return IA_ERR_UNSUPPORTED;
  const bool quads = (rot >> 1) % 4 == 0;
  const dim3 grid((unsigned)nh, (unsigned)num_tiles);
  const size_t adds_lds = sizeof(float) * RET_TILE * ret_stride(dim) + 2 * (size_t)RET_TILE * ret_vstride(vdim);
  const size_t rows_lds = ret_rows_lds(dim, vdim);
#define IA_RC_BIG(K, LDS)                                                                                                \
  do {                                                                                                                   \
    static bool allowed = false;                                                                                         \
    if ((LDS) > 60 * 1024 && !allowed) {                                                                                 \
      hipError_t e = hipFuncSetAttribute((const void*)(K), hipFuncAttributeMaxDynamicSharedMemorySize, 152 * 1024);       \
      if (e != hipSuccess) return (int)e;                                                                                \
      allowed = true;                                                                                                    \
    }                                                                                                                    \
  } while (0)
  if (quads) {
    IA_RC_BIG(retention_adds_kernel<true>, adds_lds);
    retention_adds_kernel<true><<<grid, 512, adds_lds, stream>>>((const bf16_t*)proj, tiles, first_request, records, record_stride, P);
  } else {
    IA_RC_BIG(retention_adds_kernel<false>, adds_lds);
    retention_adds_kernel<false><<<grid, 512, adds_lds, stream>>>((const bf16_t*)proj, tiles, first_request, records, record_stride, P);
  }
  IA_LAUNCH_CHECK();
  const long values = ia_retention_state_floats(nh, dim, vdim);
  retention_chain_kernel<<<dim3((unsigned)((values + 255) / 256), (unsigned)num_tiles), 256, 0, stream>>>(tiles, first_request,
                                                                                                        records, record_stride, P);
  IA_LAUNCH_CHECK();
#define IA_RC(Q, RT, JOBS)                                                                                              \
  do {                                                                                                                  \
    IA_RC_BIG((retention_rows_kernel<Q, RT, JOBS>), rows_lds);                                                           \
    retention_rows_kernel<Q, RT, JOBS><<<grid, 512, rows_lds, stream>>>((const bf16_t*)proj, (bf16_t*)out, tiles,          \
                                                                        first_request, records, record_stride, P);      \
  } while (0)
#define IA_RC_Q(Q)                           \
  do {                                       \
    if (vdim > 128) IA_RC(Q, 4, 2);          \
    else if (vdim > 64) IA_RC(Q, 4, 1);      \
    else if (vdim > 32) IA_RC(Q, 2, 1);      \
    else IA_RC(Q, 1, 1);                     \
  } while (0)
  if (quads) IA_RC_Q(true);
  else IA_RC_Q(false);
#undef IA_RC_Q
#undef IA_RC
#undef IA_RC_BIG
  IA_LAUNCH_CHECK();
  return IA_OK;
}

#include "op_call.h"
IA_OP(ia_rotation_table)
IA_OP(ia_retention_step)
IA_OP(ia_retention_chunked)
