// Recurrences with one decay per head, long segments: the gated delta rule and retention in
// chunk form, as fp32 matrix products (v_mfma_f32_16x16x4_f32) over chunks of 64 rows, so
// that only one small step per chunk is sequential.
//
// With the rows of a chunk t = 0 .. 63, their log decays l_t, G_t = l_0 + .. + l_t and the
// state S before the chunk:
//   o_t = e^{G_t} S^T q_t + sum_{j <= t} e^{G_t - G_j} (q_t.k_j) w_j
//   S' = e^{G_63} S + sum_j e^{G_63 - G_j} k_j w_j^T
// where w_j = v_j for retention.  For the delta rule w solves
//   w_t = beta_t (v_t - e^{G_t} S^T k_t - sum_{j < t} e^{G_t - G_j} (k_t.k_j) w_j),
// which is linear in S: w = U - W S with (I + A) [U | W] = [beta v | beta e^G k] and A_tj =
// beta_t e^{G_t - G_j} (k_t.k_j) for j < t.
//
// Kernels:
//   delta_solve   per (chunk, head), parallel: A on the matrix units, forward substitution with
//                 one column of [U | W] per thread; leaves U, -W and e^{G_63 - G_j} k_j
//   delta_carry   per (head, 16 columns of the state), chunk after chunk: the state stays in the
//                 accumulators of four waves (16-row tiles dealt out), whose register layout is
//                 that of a right-hand operand; leaves w and every chunk's incoming state
//   state_add     retention, per (chunk, head), parallel: a chunk's own contribution to the state
//   state_carry   retention: elementwise scan over the chunks
//   chunk_out     both, per (chunk, head, 64 columns), parallel: o from the incoming state
// Sums of log decays are formed in double precision and only their differences are rounded, so
// a chunk's decay ratios are as exact as a row-by-row walk's.
//
// A chunk's workspace index is start[s] / 64 + s + its number within the segment: distinct
// for all chunks of a step, below rows / 64 + segments.  Rows of a last, partial chunk past the
// segment's end count as k = v = 0, beta = 0, l = 0.
#include <type_traits>

#include "mx_common.h"

namespace mx {

typedef float f32x4 __attribute__((ext_vector_type(4)));
constexpr int kC = 64;          // rows per chunk
constexpr int kVLD = 80;        // floats between rows of a staged [rows][64 columns] tile
constexpr int kPLD = 68;        // floats between rows of a staged [16][64] strip

__device__ __forceinline__ f32x4 mma(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

struct ChunkIn {
  const void* q;
  const void* k;
  const void* v;
  long q_stride, k_stride, v_stride;   // elements between rows
  int rep;                             // heads per q / k head
  const float* lg;                     // log decays [T, heads], null: log_decay per head
  const double* log_decay;             // [heads]
  const float* table;                  // rotation of q and k, null: none
  int table_rows, rot_dims, interleaved;
  float k_scale;
};

// four consecutive entries as fp32 (16- or 8-byte load)
__device__ __forceinline__ void load4(const float* p, float* v) {
  const float4 u = *reinterpret_cast<const float4*>(p);
  v[0] = u.x; v[1] = u.y; v[2] = u.z; v[3] = u.w;
}
__device__ __forceinline__ void load4(const bf16_t* p, float* v) {
  const uint2 u = *reinterpret_cast<const uint2*>(p);
  ft::unpack2(u.x, v[0], v[1]);
  ft::unpack2(u.y, v[2], v[3]);
}

// rows [0, cnt) of one head of q or k into LDS [kC][LDK], rotated, times scale; zeros past cnt
// and past dk (up to DKP)
template <typename T, int DKP>
__device__ __forceinline__ void stage_head(float* dst, int LDK, const T* src, long stride, int cnt, int dk,
                                           const float* table, int table_rows, int rot, int interleaved, int pos,
                                           float scale, int vec) {
  const int tid = threadIdx.x;
  int d0 = 0;                       // entries below are rotated pairs
  if (table != nullptr && rot > 0) {
    d0 = rot;
    const int half = rot / 2;
    for (int e = tid; e < kC * half; e += 256) {
      const int t = e / half, i = e % half;
      float u = 0.f, w = 0.f;
      const int a = interleaved ? 2 * i : i, b = interleaved ? 2 * i + 1 : i + half;
      if (t < cnt) {
        int p = pos + t;
        if (p < 0 || p >= table_rows) p = 0;
        const float c = table[(long)p * rot + i], sn = table[(long)p * rot + half + i];
        const float x = ld(src, t * stride + a), y = ld(src, t * stride + b);
        u = (x * c - y * sn) * scale;
        w = (y * c + x * sn) * scale;
      }
      dst[t * LDK + a] = u;
      dst[t * LDK + b] = w;
    }
  }
  if (vec && d0 == 0) {
    for (int e = tid; e < kC * (DKP / 4); e += 256) {
      const int t = e / (DKP / 4), i = e % (DKP / 4) * 4;
      float v[4] = {0.f, 0.f, 0.f, 0.f};
      if (t < cnt && i < dk) load4(src + t * stride + i, v);
#pragma unroll
      for (int j = 0; j < 4; ++j) dst[t * LDK + i + j] = v[j] * scale;
    }
    return;
  }
  const int rest = DKP - d0;
  if (rest <= 0) return;
  for (int e = tid; e < kC * rest; e += 256) {
    const int t = e / rest, i = d0 + e % rest;
    dst[t * LDK + i] = t < cnt && i < dk ? ld(src, t * stride + i) * scale : 0.f;
  }
}

// rows [0, cnt) x 64 columns from col0 of a [., dv] array into LDS [kC][kVLD], zeros elsewhere
template <typename T>
__device__ __forceinline__ void stage_cols(float* dst, const T* src, long stride, int cnt, int col0, int dv, int vec) {
  const int tid = threadIdx.x;
  if (vec) {
    for (int e = tid; e < kC * 16; e += 256) {
      const int t = e >> 4, c = (e & 15) * 4;
      float v[4] = {0.f, 0.f, 0.f, 0.f};
      if (t < cnt && col0 + c < dv) load4(src + t * stride + col0 + c, v);
      *reinterpret_cast<float4*>(dst + t * kVLD + c) = make_float4(v[0], v[1], v[2], v[3]);
    }
  } else {
    for (int e = tid; e < kC * 64; e += 256) {
      const int t = e >> 6, c = e & 63;
      dst[t * kVLD + c] = t < cnt && col0 + c < dv ? ld(src, t * stride + col0 + c) : 0.f;
    }
  }
}

// G[t] = sum of the chunk's log decays up to t (wave 0; 64 rows)
__device__ __forceinline__ void stage_log_decay(double* G, const ChunkIn& in, long row0, int cnt, int heads, int h) {
  if (threadIdx.x >= 64) return;
  const int t = threadIdx.x;
  double l = 0.0;
  if (t < cnt) l = in.lg != nullptr ? (double)in.lg[(row0 + t) * heads + h] : in.log_decay[h];
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const double u = __shfl_up(l, off, 64);
    if (t >= off) l += u;
  }
  G[t] = l;
}

// the chunk of this workgroup: false if the segment has no such chunk (or is left to the walk)
struct Chunk {
  int cnt, num, pos, slot;
  long row0, ws;
};
__device__ __forceinline__ bool find_chunk(Chunk& c, int idx, int s, const int* start, const int* pos0, const int* slot,
                                           int min_rows, int num_slots) {
  const int r0 = start[s], n = start[s + 1] - r0;
  c.slot = slot[s];
  if (n < min_rows || n <= 0 || c.slot < 0 || c.slot >= num_slots) return false;
  c.num = (n + kC - 1) / kC;
  if (idx >= c.num) return false;
  c.cnt = min(kC, n - idx * kC);
  c.row0 = r0 + (long)idx * kC;
  c.pos = pos0[s] + idx * kC;
  c.ws = r0 / kC + s + idx;
  return true;
}

// ---------------------------------------------------------------------------------
// grid (chunks, heads * ceil(dv / 64), segments): L = sum_j e^{G_last - G_j} k_j v_j^T into the
// chunk's workspace [dk, dv].  Wave w: columns 16 w .. 16 w + 15 of the 64, all rows.
// ---------------------------------------------------------------------------------
template <typename T, int DKT>
__global__ void __launch_bounds__(256)
state_add_kernel(float* __restrict__ ws_s, ChunkIn in, const int* __restrict__ start, const int* __restrict__ pos0,
                 const int* __restrict__ slot, int heads, int dk, int dv, int num_slots, int min_rows, int vec) {
  constexpr int DKP = 16 * DKT, LDK = DKP + 16;
  __shared__ __attribute__((aligned(16))) float kb[kC * LDK], vb[kC * kVLD];
  __shared__ double G[kC];
  Chunk c;
  if (!find_chunk(c, blockIdx.x, blockIdx.z, start, pos0, slot, min_rows, num_slots)) return;
  const int vt = (dv + 63) / 64;
  const int h = blockIdx.y / vt, col0 = blockIdx.y % vt * 64;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lo = lane & 15, hi = lane >> 4;
  stage_log_decay(G, in, c.row0, c.cnt, heads, h);
  stage_head<T, DKP>(kb, LDK, (const T*)in.k + c.row0 * in.k_stride + (long)(h / in.rep) * dk, in.k_stride, c.cnt, dk,
                     in.table, in.table_rows, in.rot_dims, in.interleaved, c.pos, in.k_scale, vec);
  stage_cols<T>(vb, (const T*)in.v + c.row0 * in.v_stride + (long)h * dv, in.v_stride, c.cnt, col0, dv, vec);
  __syncthreads();
  const double gl = G[kC - 1];
  f32x4 acc[DKT];
#pragma unroll
  for (int i = 0; i < DKT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int s = 0; s < kC / 4; ++s) {
    const int j = 4 * s + hi;
    const float b = vb[j * kVLD + 16 * wave + lo] * expf((float)(gl - G[j]));
#pragma unroll
    for (int i = 0; i < DKT; ++i) acc[i] = mma(kb[j * LDK + 16 * i + lo], b, acc[i]);
  }
  const int col = col0 + 16 * wave + lo;
  if (col >= dv) return;
  float* out = ws_s + ((c.ws * heads + h) * dk) * dv + col;
#pragma unroll
  for (int i = 0; i < DKT; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = 16 * i + 4 * hi + r;
      if (row < dk) out[(long)row * dv] = acc[i][r];
    }
}

// grid (ceil(dk dv / 256), heads, segments): workspaces hold every chunk's own contribution L_c
// and become its incoming state; the last one goes to the slot
__global__ void __launch_bounds__(256)
state_carry_kernel(float* __restrict__ ws_s, const double* __restrict__ log_decay, float* __restrict__ state,
                   const int* __restrict__ start, const int* __restrict__ pos0, const int* __restrict__ slot, int heads,
                   int size, int num_slots, int min_rows) {
  Chunk c;
  if (!find_chunk(c, 0, blockIdx.z, start, pos0, slot, min_rows, num_slots)) return;
  const int h = blockIdx.y, e = blockIdx.x * 256 + threadIdx.x;
  if (e >= size) return;
  const int n = start[blockIdx.z + 1] - start[blockIdx.z];
  float* sp = state + ((long)c.slot * heads + h) * size + e;
  float S = c.pos > 0 ? *sp : 0.f;
  const float full = (float)exp(log_decay[h] * kC), last = (float)exp(log_decay[h] * (n - (c.num - 1) * kC));
  float* w = ws_s + (c.ws * heads + h) * (long)size + e;
  const long step = (long)heads * size;
  constexpr int AHEAD = 8;            // contributions in flight
  for (int i0 = 0; i0 < c.num; i0 += AHEAD) {
    float l[AHEAD];
#pragma unroll
    for (int u = 0; u < AHEAD; ++u) l[u] = i0 + u < c.num ? w[(i0 + u) * step] : 0.f;
#pragma unroll
    for (int u = 0; u < AHEAD; ++u) {
      if (i0 + u < c.num) {
        w[(i0 + u) * step] = S;
        S = (i0 + u + 1 < c.num ? full : last) * S + l[u];
      }
    }
  }
  *sp = S;
}

// ---------------------------------------------------------------------------------
// grid (chunks, heads * ceil(dv / 64), segments): o of the chunk's rows.  Wave w: rows 16 w ..
// 16 w + 15, 64 columns; its q rows stay in registers as left-hand operands.
// ---------------------------------------------------------------------------------
template <typename T, int DKT>
__global__ void __launch_bounds__(256)
chunk_out_kernel(float* __restrict__ o, ChunkIn in, const float* __restrict__ ws_s, const int* __restrict__ start,
                 const int* __restrict__ pos0, const int* __restrict__ slot, int heads, int dk, int dv, int num_slots,
                 int min_rows, int vec) {
  constexpr int DKP = 16 * DKT, LDK = DKP + 4;
  constexpr int KB = kC * LDK > 64 * kPLD ? kC * LDK : 64 * kPLD;
  __shared__ __attribute__((aligned(16))) float kb[KB], vb[kC * kVLD];
  __shared__ double G[kC];
  const int vt = (dv + 63) / 64;
  const int h = blockIdx.y / vt, col0 = blockIdx.y % vt * 64;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lo = lane & 15, hi = lane >> 4;
  Chunk c;
  if (!find_chunk(c, blockIdx.x, blockIdx.z, start, pos0, slot, min_rows, num_slots)) {
    // a padding segment's rows are zeros
    const int s = blockIdx.z, r0 = start[s], n = start[s + 1] - r0;
    if (n >= min_rows && (slot[s] < 0 || slot[s] >= num_slots))
      for (int e = tid; e < kC * 64; e += 256) {
        const int t = blockIdx.x * kC + (e >> 6), cc = col0 + (e & 63);
        if (t < n && cc < dv) o[((long)(r0 + t) * heads + h) * dv + cc] = 0.f;
      }
    return;
  }
  const long hoff = (long)(h / in.rep) * dk;
  const float* S = ws_s + ((c.ws * heads + h) * dk) * (long)dv;
  stage_log_decay(G, in, c.row0, c.cnt, heads, h);
  stage_head<T, DKP>(kb, LDK, (const T*)in.q + c.row0 * in.q_stride + hoff, in.q_stride, c.cnt, dk, in.table,
                     in.table_rows, in.rot_dims, in.interleaved, c.pos, 1.f, vec);
  const int svec = dv % 4 == 0;
  stage_cols<float>(vb, S, dv, dk, col0, dv, svec);         // rows 0 .. 63 of the incoming state
  __syncthreads();
  float qf[4 * DKT];
#pragma unroll
  for (int s = 0; s < 4 * DKT; ++s) qf[s] = kb[(16 * wave + lo) * LDK + 4 * s + hi];
  f32x4 O[4];
#pragma unroll
  for (int ct = 0; ct < 4; ++ct) O[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < (DKT < 4 ? 4 * DKT : 16); ++s)
#pragma unroll
    for (int ct = 0; ct < 4; ++ct) O[ct] = mma(qf[s], vb[(4 * s + hi) * kVLD + 16 * ct + lo], O[ct]);
  __syncthreads();
  if constexpr (DKT > 4) {                                   // rows 64 .. of the state
    stage_cols<float>(vb, S + 64L * dv, dv, dk - 64, col0, dv, svec);
    __syncthreads();
#pragma unroll
    for (int s = 16; s < 4 * DKT; ++s)
#pragma unroll
      for (int ct = 0; ct < 4; ++ct) O[ct] = mma(qf[s], vb[(4 * (s - 16) + hi) * kVLD + 16 * ct + lo], O[ct]);
    __syncthreads();
  }
  stage_head<T, DKP>(kb, LDK, (const T*)in.k + c.row0 * in.k_stride + hoff, in.k_stride, c.cnt, dk, in.table,
                     in.table_rows, in.rot_dims, in.interleaved, c.pos, in.k_scale, vec);
  stage_cols<T>(vb, (const T*)in.v + c.row0 * in.v_stride + (long)h * dv, in.v_stride, c.cnt, col0, dv, vec);
  double gr[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    gr[r] = G[16 * wave + 4 * hi + r];
    const float e = expf((float)gr[r]);
#pragma unroll
    for (int ct = 0; ct < 4; ++ct) O[ct][r] *= e;
  }
  __syncthreads();
  f32x4 P[4];
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
    if (jt > wave) continue;                                 // keys behind every row of this wave
    f32x4 a = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < 4 * DKT; ++s) a = mma(qf[s], kb[(16 * jt + lo) * LDK + 4 * s + hi], a);
    const double gj = G[16 * jt + lo];
#pragma unroll
    for (int r = 0; r < 4; ++r)
      a[r] = 16 * jt + lo <= 16 * wave + 4 * hi + r ? a[r] * expf((float)(gr[r] - gj)) : 0.f;
    P[jt] = a;
  }
  __syncthreads();                                           // kb becomes four [16][64] strips
  float* strip = kb + wave * 16 * kPLD;
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
    if (jt > wave) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r) strip[(4 * hi + r) * kPLD + 16 * jt + lo] = P[jt][r];
  }
  wave_lds_fence();
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
    if (jt > wave) continue;
#pragma unroll
    for (int s = 4 * jt; s < 4 * jt + 4; ++s) {
      const float a = strip[lo * kPLD + 4 * s + hi];
#pragma unroll
      for (int ct = 0; ct < 4; ++ct) O[ct] = mma(a, vb[(4 * s + hi) * kVLD + 16 * ct + lo], O[ct]);
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int t = 16 * wave + 4 * hi + r;
    if (t >= c.cnt) continue;
    float* op = o + ((c.row0 + t) * heads + h) * dv;
#pragma unroll
    for (int ct = 0; ct < 4; ++ct)
      if (col0 + 16 * ct + lo < dv) op[col0 + 16 * ct + lo] = O[ct][r];
  }
}

// ---------------------------------------------------------------------------------
// grid (chunks, heads, segments), 256 threads.  Leaves per chunk and head: -W [64][DKP],
// (e^{G_last - G_j} k_j)^T [DKP][64], e^{G_last}; and U in rows [T, heads, dv].
// ---------------------------------------------------------------------------------
template <int DKT>
__global__ void __launch_bounds__(256)
delta_solve_kernel(float* __restrict__ ws_w, float* __restrict__ ws_k, float* __restrict__ ws_u,
                   float* __restrict__ ws_g, ChunkIn in, const float* __restrict__ beta, const int* __restrict__ start,
                   const int* __restrict__ pos0, const int* __restrict__ slot, int heads, int dk, int dv, int num_slots,
                   int min_rows, int vec) {
  constexpr int DKP = 16 * DKT, LDK = DKP + 4;
  // A transposed: at[j][i] = A_ij, so that the substitution reads the rows below j together
  __shared__ __attribute__((aligned(16))) float kb[kC * LDK], at[kC * kPLD];
  __shared__ double G[kC];
  __shared__ float bs[kC], eg[kC], el[kC];
  Chunk c;
  if (!find_chunk(c, blockIdx.x, blockIdx.z, start, pos0, slot, min_rows, num_slots)) return;
  const int h = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lo = lane & 15, hi = lane >> 4;
  stage_log_decay(G, in, c.row0, c.cnt, heads, h);
  if (tid >= 64 && tid < 128) bs[tid - 64] = tid - 64 < c.cnt ? beta[(c.row0 + tid - 64) * heads + h] : 0.f;
  stage_head<float, DKP>(kb, LDK, (const float*)in.k + c.row0 * in.k_stride + (long)(h / in.rep) * dk, in.k_stride, c.cnt,
                         dk, nullptr, 0, 0, 0, 0, 1.f, vec);
  __syncthreads();
  if (tid < kC) {
    eg[tid] = expf((float)G[tid]);
    el[tid] = expf((float)(G[kC - 1] - G[tid]));
    if (tid == 0) ws_g[c.ws * heads + h] = expf((float)G[kC - 1]);
  }
  {
    float kf[4 * DKT];
#pragma unroll
    for (int s = 0; s < 4 * DKT; ++s) kf[s] = kb[(16 * wave + lo) * LDK + 4 * s + hi];
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      if (jt > wave) continue;
      f32x4 a = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < 4 * DKT; ++s) a = mma(kf[s], kb[(16 * jt + lo) * LDK + 4 * s + hi], a);
      const int j = 16 * jt + lo;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * wave + 4 * hi + r;
        at[j * kPLD + i] = j < i ? bs[i] * a[r] * expf((float)(G[i] - G[j])) : 0.f;
      }
    }
  }
  __syncthreads();
  float* wk = ws_k + (c.ws * heads + h) * (long)DKP * kC;
  for (int e = tid; e < DKP * kC; e += 256) {
    const int d = e / kC, j = e % kC;
    wk[e] = kb[j * LDK + d] * el[j];
  }
  float* ww = ws_w + (c.ws * heads + h) * (long)kC * DKP;
  for (int col = tid; col < DKP + dv; col += 256) {
    const bool is_w = col < DKP;
    float x[kC];
    if (is_w) {
#pragma unroll
      for (int i = 0; i < kC; ++i) x[i] = bs[i] * eg[i] * kb[i * LDK + col];
    } else {
      const float* vp = (const float*)in.v + c.row0 * in.v_stride + (long)h * dv + (col - DKP);
#pragma unroll
      for (int i = 0; i < kC; ++i) x[i] = i < c.cnt ? bs[i] * vp[i * in.v_stride] : 0.f;
    }
#pragma unroll
    for (int j = 0; j < kC - 1; ++j) {
      const float xj = x[j];
#pragma unroll
      for (int i4 = (j + 1) / 4; i4 < kC / 4; ++i4) {
        const float4 a = *reinterpret_cast<const float4*>(&at[j * kPLD + 4 * i4]);
        const float av[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
        for (int u = 0; u < 4; ++u)
          if (4 * i4 + u > j) x[4 * i4 + u] -= av[u] * xj;
      }
    }
    if (is_w) {
#pragma unroll
      for (int i = 0; i < kC; ++i) ww[(long)i * DKP + col] = -x[i];
    } else {
#pragma unroll
      for (int i = 0; i < kC; ++i)
        if (i < c.cnt) ws_u[((c.row0 + i) * heads + h) * dv + (col - DKP)] = x[i];
    }
  }
}

// ---------------------------------------------------------------------------------
// grid (ceil(dv / 16), heads, segments), four waves: the state's 16 columns, chunk after chunk.
// Wave w holds the 16-row tiles w IT .. w IT + IT - 1 in accumulators; accumulator register r of
// lane (hi, lo) is row 4 hi + r, column lo, which is also a right-hand operand whose inner index
// 4 hi + r the left-hand operands (16-byte loads) follow.  Per chunk: every wave's part of
// -W S for all 64 rows, the parts added through LDS (wave w adds U and owns rows 16 w ..), w left
// in place of U, then S <- e^{G_last} S + K^T w.  Two register sets keep a chunk's operands
// on their way while the chunk before is computed.
// ---------------------------------------------------------------------------------
template <int DKT>
__global__ void __launch_bounds__(256)
delta_carry_kernel(float* __restrict__ ws_s, const float* __restrict__ ws_w, const float* __restrict__ ws_k,
                   float* __restrict__ ws_u, const float* __restrict__ ws_g, float* __restrict__ state,
                   const int* __restrict__ start, const int* __restrict__ pos0, const int* __restrict__ slot, int heads,
                   int dk, int dv, int num_slots, int min_rows) {
  constexpr int DKP = 16 * DKT, IT = DKT < 4 ? 1 : DKT / 4;
  __shared__ f32x4 part[4][4][64], whole[4][64];
  Chunk c;
  if (!find_chunk(c, 0, blockIdx.z, start, pos0, slot, min_rows, num_slots)) return;
  const int h = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lo = lane & 15, hi = lane >> 4;
  const int n = start[blockIdx.z + 1] - start[blockIdx.z];
  const int col = blockIdx.x * 16 + lo;
  const bool live = col < dv;
  const bool mine = wave * IT < DKT;                 // few tiles: some waves only add
  float* sp = state + (((long)c.slot * heads + h) * dk) * dv + col;
  f32x4 S[IT];
#pragma unroll
  for (int ii = 0; ii < IT; ++ii)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = 16 * (wave * IT + ii) + 4 * hi + r;
      S[ii][r] = c.pos > 0 && mine && live && row < dk ? sp[(long)row * dv] : 0.f;
    }
  struct Ops {
    f32x4 w[4][IT], k[IT][4], u;
    float g;
  };
  auto fetch = [&](Ops& f, int idx) {
    if (idx >= c.num) return;
    const long cs = (c.ws + idx) * heads + h;
    const float* w = ws_w + cs * kC * DKP;
    const float* k = ws_k + cs * DKP * kC;
    if (mine) {
#pragma unroll
      for (int m = 0; m < 4; ++m)
#pragma unroll
        for (int ii = 0; ii < IT; ++ii) {
          const int i = wave * IT + ii;
          f.w[m][ii] = *reinterpret_cast<const f32x4*>(w + (16 * m + lo) * DKP + 16 * i + 4 * hi);
          f.k[ii][m] = *reinterpret_cast<const f32x4*>(k + (16 * i + lo) * kC + 16 * m + 4 * hi);
        }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = idx * kC + 16 * wave + 4 * hi + r;
      f.u[r] = t < n && live ? ws_u[((c.row0 + t) * heads + h) * dv + col] : 0.f;
    }
    f.g = ws_g[cs];
  };
  auto turn = [&](const Ops& f, int idx) {
    float* so = ws_s + (((c.ws + idx) * heads + h) * dk) * (long)dv + col;
    if (mine && live) {
#pragma unroll
      for (int ii = 0; ii < IT; ++ii)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int row = 16 * (wave * IT + ii) + 4 * hi + r;
          if (row < dk) so[(long)row * dv] = S[ii][r];
        }
    }
#pragma unroll
    for (int m = 0; m < 4; ++m) {
      f32x4 a = f32x4{0.f, 0.f, 0.f, 0.f};
      if (mine) {
#pragma unroll
        for (int ii = 0; ii < IT; ++ii)
#pragma unroll
          for (int r = 0; r < 4; ++r) a = mma(f.w[m][ii][r], S[ii][r], a);
      }
      part[m][wave][lane] = a;
    }
    __syncthreads();
    f32x4 v = f.u;
#pragma unroll
    for (int w = 0; w < 4; ++w) v += part[wave][w][lane];
    whole[wave][lane] = v;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = idx * kC + 16 * wave + 4 * hi + r;
      if (t < n && live) ws_u[((c.row0 + t) * heads + h) * dv + col] = v[r];
    }
    __syncthreads();
    if (mine) {
#pragma unroll
      for (int ii = 0; ii < IT; ++ii) S[ii] *= f.g;
#pragma unroll
      for (int m = 0; m < 4; ++m) {
        const f32x4 vm = whole[m][lane];
#pragma unroll
        for (int ii = 0; ii < IT; ++ii)
#pragma unroll
          for (int r = 0; r < 4; ++r) S[ii] = mma(f.k[ii][m][r], vm[r], S[ii]);
      }
    }
  };
  Ops fa, fb;
  fetch(fa, 0);
  fetch(fb, 1);
  for (int idx = 0; idx < c.num; idx += 2) {
    turn(fa, idx);
    fetch(fa, idx + 2);
    if (idx + 1 >= c.num) break;
    turn(fb, idx + 1);
    fetch(fb, idx + 3);
  }
  if (mine && live) {
#pragma unroll
    for (int ii = 0; ii < IT; ++ii)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = 16 * (wave * IT + ii) + 4 * hi + r;
        if (row < dk) sp[(long)row * dv] = S[ii][r];
      }
  }
}

}  // namespace mx

using namespace mx;

extern "C" int mx_chunk_rows() { return kC; }
extern "C" int mx_chunk_max_dk() { return 128; }
// key size up to the kernels' whole tiles (rows of the -W and key workspaces)
extern "C" int mx_chunk_key_pad(int dk) { return dk <= 16 ? 16 : dk <= 32 ? 32 : dk <= 64 ? 64 : 128; }

// calls f with the key size's tile count as a constant
template <typename F>
static void key_tiles(int dk, F f) {
  const int t = (dk + 15) / 16;
  if (t <= 1) f(std::integral_constant<int, 1>{});
  else if (t <= 2) f(std::integral_constant<int, 2>{});
  else if (t <= 4) f(std::integral_constant<int, 4>{});
  else f(std::integral_constant<int, 8>{});
}

template <typename T>
static void launch_out(float* o, const ChunkIn& in, const float* ws_s, const int* start, const int* pos0,
                       const int* slot, dim3 grid, int heads, int dk, int dv, int num_slots, int min_rows, int vec,
                       hipStream_t s) {
  key_tiles(dk, [&](auto t) {
    hipLaunchKernelGGL((chunk_out_kernel<T, decltype(t)::value>), grid, dim3(256), 0, s, o, in, ws_s, start, pos0, slot,
                       heads, dk, dv, num_slots, min_rows, vec);
  });
}

extern "C" int mx_retention_chunks(float* o, const void* p, int bf16, long stride, const float* table, int table_rows,
                                   int rot_dims, int interleaved, const double* log_decay, float* state, float* ws_s,
                                   const int* start, const int* pos0, const int* slot, int num_segs, int max_rows,
                                   int heads, int dk, int dv, int num_slots, int min_rows, hipStream_t s) {
  if (num_segs <= 0 || max_rows < min_rows) return 0;
  if (dk < 1 || dk > mx_chunk_max_dk() || dv < 1 || heads < 1 || min_rows < 1) return -1;
  ChunkIn in{};
  const long es = bf16 ? 2 : 4;
  in.q = p;
  in.k = (const char*)p + es * heads * dk;
  in.v = (const char*)p + es * 2 * heads * dk;
  in.q_stride = in.k_stride = in.v_stride = stride;
  in.rep = 1;
  in.log_decay = log_decay;
  in.table = rot_dims > 0 ? table : nullptr;
  in.table_rows = table_rows; in.rot_dims = rot_dims; in.interleaved = interleaved;
  in.k_scale = 1.0f / sqrtf((float)dk);
  const int vec = dk % 4 == 0 && dv % 4 == 0 && stride % 4 == 0 && ((uintptr_t)p) % (4 * es) == 0;
  const dim3 grid((max_rows + kC - 1) / kC, heads * ((dv + 63) / 64), num_segs);
  if (grid.y > 65535 || grid.z > 65535) return -2;
  MX_DISPATCH_T(bf16, key_tiles(dk, [&](auto t) {
    hipLaunchKernelGGL((state_add_kernel<T, decltype(t)::value>), grid, dim3(256), 0, s, ws_s, in, start, pos0, slot,
                       heads, dk, dv, num_slots, min_rows, vec);
  }));
  hipLaunchKernelGGL(state_carry_kernel, dim3((dk * dv + 255) / 256, heads, num_segs), dim3(256), 0, s, ws_s, log_decay,
                     state, start, pos0, slot, heads, dk * dv, num_slots, min_rows);
  MX_DISPATCH_T(bf16, (launch_out<T>(o, in, ws_s, start, pos0, slot, grid, heads, dk, dv, num_slots, min_rows, vec, s)));
  return (int)hipGetLastError();
}

extern "C" int mx_head_delta_chunks(float* o, const float* q, const float* k, const float* v, const float* lg,
                                    const float* beta, float* state, float* ws_s, float* ws_w, float* ws_k, float* ws_u,
                                    float* ws_g, const int* start, const int* pos0, const int* slot, int num_segs,
                                    int max_rows, int heads, int kv_heads, int dk, int dv, int num_slots, int min_rows,
                                    hipStream_t s) {
  if (num_segs <= 0 || max_rows < min_rows) return 0;
  if (dk < 1 || dk > mx_chunk_max_dk() || dv < 1 || kv_heads < 1 || heads % kv_heads || min_rows < 1) return -1;
  ChunkIn in{};
  in.q = q; in.k = k; in.v = v;
  in.q_stride = in.k_stride = (long)kv_heads * dk;
  in.v_stride = (long)heads * dv;
  in.rep = heads / kv_heads;
  in.lg = lg;
  in.k_scale = 1.f;
  const int vec = dk % 4 == 0 && dv % 4 == 0 && (((uintptr_t)q | (uintptr_t)k | (uintptr_t)v | (uintptr_t)ws_u) % 16) == 0;
  const int chunks = (max_rows + kC - 1) / kC;
  if (heads > 65535 || (long)heads * ((dv + 63) / 64) > 65535 || num_segs > 65535) return -2;
  key_tiles(dk, [&](auto t) {
    hipLaunchKernelGGL((delta_solve_kernel<decltype(t)::value>), dim3(chunks, heads, num_segs), dim3(256), 0, s, ws_w,
                       ws_k, ws_u, ws_g, in, beta, start, pos0, slot, heads, dk, dv, num_slots, min_rows, vec);
    hipLaunchKernelGGL((delta_carry_kernel<decltype(t)::value>), dim3((dv + 15) / 16, heads, num_segs), dim3(256), 0, s,
                       ws_s, ws_w, ws_k, ws_u, ws_g, state, start, pos0, slot, heads, dk, dv, num_slots, min_rows);
  });
  in.v = ws_u;                     // the solved rows take the values' place
  launch_out<float>(o, in, ws_s, start, pos0, slot, dim3(chunks, heads * ((dv + 63) / 64), num_segs), heads, dk, dv,
                    num_slots, min_rows, vec, s);
  return (int)hipGetLastError();
}
