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
//   delta_solve   per (chunk, head), parallel: A, (I + A)^-1 (16-row diagonal blocks by
//                 substitution, the rest by block products) and [U | W] on the matrix units;
//                 leaves U, -W and e^{G_63 - G_j} k_j.  (The inverse is harmless numerically:
//                 its entries are -beta k^T (products of I - beta k k^T) k, at most one in size.)
//   delta_carry   per (head, 16 columns of the state), chunk after chunk: the state stays in the
//                 accumulators of four waves (16-row tiles dealt out), whose register layout is
//                 that of a right-hand operand; leaves w and every chunk's incoming state
//   state_add     retention, per (chunk, head), parallel: a chunk's own contribution to the state
//   state_carry   retention: elementwise scan over the chunks
//   chunk_out     both, per (chunk, head, 64 columns), parallel: o from the incoming state
// Sums of log decays are formed in double precision and only their differences are rounded, so
// a chunk's decay ratios are as exact as a row-by-row walk's.
//
// delta_solve leaves -W, the keys and U as fragments: for every 16 x 16 tile one 16-byte piece per
// lane (hi, lo) = (lane / 16, lane % 16), in the lanes' order, so that delta_carry's operand
// loads are whole kilobytes: -W tile (m, i) holds rows 16 m + lo, columns 16 i + 4 hi + r; key
// tile (i, m) columns 16 i + lo, rows 16 m + 4 hi + r; U tile (ct, m) rows 16 m + 4 hi + r, column
// 16 ct + lo (r = 0 .. 3 the piece's entries).
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

// a product over N inner steps of 4, a(s) and b(s) the operands of step s: four sums in turn, so
// that no product waits for the one before
template <int N, typename A, typename B>
__device__ __forceinline__ f32x4 dot_steps(A a, B b) {
  f32x4 p[4];
#pragma unroll
  for (int u = 0; u < 4; ++u) p[u] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < N; ++s) p[s & 3] = mma(a(s), b(s), p[s & 3]);
  return (p[0] + p[1]) + (p[2] + p[3]);
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
  int v_frags;                         // v: fragments by workspace chunk (below) instead of rows
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
  const int t0 = tid >> 5, l0 = tid & 31;   // without 16-byte pieces: 32 lanes per row, 8 rows at a time
  int d0 = 0;                       // entries below are rotated pairs
  if (table != nullptr && rot > 0) {
    d0 = rot;
    const int half = rot / 2;
#pragma unroll 4
    for (int t = t0; t < kC; t += 8) {
      // rows past cnt read the last row and count as zeros
      const int tt = min(t, cnt - 1);
      int p = pos + tt;
      if (p < 0 || p >= table_rows) p = 0;
      const float* cs = table + (long)p * rot;
      const float f = t < cnt ? scale : 0.f;
      for (int i = l0; i < half; i += 32) {
        const int a = interleaved ? 2 * i : i, b = interleaved ? 2 * i + 1 : i + half;
        const float c = cs[i], sn = cs[half + i];
        const float x = ld(src, tt * stride + a), y = ld(src, tt * stride + b);
        dst[t * LDK + a] = (x * c - y * sn) * f;
        dst[t * LDK + b] = (y * c + x * sn) * f;
      }
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
  for (int t = t0; t < kC; t += 8)
    for (int i = d0 + l0; i < DKP; i += 32) dst[t * LDK + i] = t < cnt && i < dk ? ld(src, t * stride + i) * scale : 0.f;
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
  if (in.v_frags) {
    const int tiles = (dv + 15) / 16;
    const float4* fp = (const float4*)in.v + (c.ws * heads + h) * (long)tiles * 256;
    for (int ct = wave; ct < 4; ct += 4) {
      const int tile = min(col0 / 16 + ct, tiles - 1);       // columns past dv are not stored
#pragma unroll
      for (int m = 0; m < 4; ++m) {
        const float4 u = fp[(tile * 4 + m) * 64 + lane];
        const float v[4] = {u.x, u.y, u.z, u.w};
#pragma unroll
        for (int r = 0; r < 4; ++r) vb[(16 * m + 4 * hi + r) * kVLD + 16 * ct + lo] = v[r];
      }
    }
  } else {
    stage_cols<T>(vb, (const T*)in.v + c.row0 * in.v_stride + (long)h * dv, in.v_stride, c.cnt, col0, dv, vec);
  }
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
    const float* kr = kb + (16 * jt + lo) * LDK + hi;
    f32x4 a = dot_steps<4 * DKT>([&](int s) { return qf[s]; }, [&](int s) { return kr[4 * s]; });
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
// grid (chunks, heads, segments), 256 threads.  Leaves per chunk and head, as fragments: -W,
// e^{G_last - G_j} k_j and U; and e^{G_last}.
// ---------------------------------------------------------------------------------
template <int DKT>
__global__ void __launch_bounds__(256)
delta_solve_kernel(float* __restrict__ ws_w, float* __restrict__ ws_k, float* __restrict__ ws_u,
                   float* __restrict__ ws_g, ChunkIn in, const float* __restrict__ beta, const int* __restrict__ start,
                   const int* __restrict__ pos0, const int* __restrict__ slot, int heads, int dk, int dv, int num_slots,
                   int min_rows, int vec) {
  constexpr int DKP = 16 * DKT, LDK = DKP + 4;
  // ab: A, block by block replaced by T = (I + A)^-1 (blocks above the diagonal are never read)
  __shared__ __attribute__((aligned(16))) float kb[kC * LDK], ab[kC * kPLD];
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
    eg[tid] = expf((float)G[tid]) * bs[tid];
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
      const float* kr = kb + (16 * jt + lo) * LDK + hi;
      const f32x4 a = dot_steps<4 * DKT>([&](int s) { return kf[s]; }, [&](int s) { return kr[4 * s]; });
      const int j = 16 * jt + lo;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * wave + 4 * hi + r;
        ab[i * kPLD + j] = j < i ? bs[i] * a[r] * expf((float)(G[i] - G[j])) : 0.f;
      }
    }
  }
  wave_lds_fence();
  {
    // the wave's own diagonal block: lane lo holds column lo of its inverse (the four quarters
    // of the wave do the same work)
    float* d = ab + 16 * wave * kPLD + 16 * wave;
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) x[i] = i == lo ? 1.f : 0.f;
#pragma unroll
    for (int j = 0; j < 15; ++j)
#pragma unroll
      for (int i = j + 1; i < 16; ++i) x[i] -= d[i * kPLD + j] * x[j];
    wave_lds_fence();
    if (hi == 0) {
#pragma unroll
      for (int i = 0; i < 16; ++i) d[i * kPLD + lo] = x[i];
    }
  }
  __syncthreads();
  // below the diagonal, one row of blocks after the other: T_ij = -T_ii sum_{j <= k < i} A_ik T_kj
#pragma unroll
  for (int i = 1; i < 4; ++i) {
    f32x4 t = f32x4{0.f, 0.f, 0.f, 0.f};
    const int j = wave;
    if (j < i) {
      f32x4 m = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < i; ++k) {
        if (k < j) continue;
#pragma unroll
        for (int s = 0; s < 4; ++s)
          m = mma(ab[(16 * i + lo) * kPLD + 16 * k + 4 * s + hi], ab[(16 * k + 4 * s + hi) * kPLD + 16 * j + lo], m);
      }
      // m in accumulator layout is a right-hand operand with inner index 4 hi + r
#pragma unroll
      for (int r = 0; r < 4; ++r) t = mma(-ab[(16 * i + lo) * kPLD + 16 * i + 4 * hi + r], m[r], t);
    }
    __syncthreads();
    if (j < i) {
#pragma unroll
      for (int r = 0; r < 4; ++r) ab[(16 * i + 4 * hi + r) * kPLD + 16 * j + lo] = t[r];
    }
    __syncthreads();
  }
  // [W | U] = T [beta e^G k | beta v], column tiles dealt out to the waves
  float tf[4][16], fw[16], fu[16];
#pragma unroll
  for (int m = 0; m < 4; ++m)
#pragma unroll
    for (int s = 0; s < 4 * m + 4; ++s) tf[m][s] = ab[(16 * m + lo) * kPLD + 4 * s + hi];
#pragma unroll
  for (int s = 0; s < 16; ++s) {
    fw[s] = eg[4 * s + hi];
    fu[s] = bs[4 * s + hi];
  }
  // four row tiles of T b, or of its transpose (the operands in turn: their layouts are alike)
  auto column = [&](const float (&b)[16], f32x4 (&x)[4], auto transposed) {
#pragma unroll
    for (int m = 0; m < 4; ++m) x[m] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < 16; ++s)
#pragma unroll
      for (int m = s / 4; m < 4; ++m)
        x[m] = decltype(transposed)::value ? mma(b[s], tf[m][s], x[m]) : mma(tf[m][s], b[s], x[m]);
  };
  f32x4* ww = (f32x4*)ws_w + (c.ws * heads + h) * (long)(4 * DKT * 64);
  for (int ct = wave; ct < DKT; ct += 4) {
    float b[16];
    f32x4 x[4];
#pragma unroll
    for (int s = 0; s < 16; ++s) b[s] = -fw[s] * kb[(4 * s + hi) * LDK + 16 * ct + lo];
    column(b, x, std::integral_constant<bool, true>{});
#pragma unroll
    for (int m = 0; m < 4; ++m) ww[(m * DKT + ct) * 64 + lane] = x[m];
  }
  const int vtiles = (dv + 15) / 16;
  f32x4* wu = (f32x4*)ws_u + (c.ws * heads + h) * (long)vtiles * 256;
  for (int ct = wave; ct < vtiles; ct += 4) {
    float b[16];
    f32x4 x[4];
    const int col = 16 * ct + lo;
    const float* vp = (const float*)in.v + c.row0 * in.v_stride + (long)h * dv + min(col, dv - 1);
#pragma unroll
    for (int s = 0; s < 16; ++s) b[s] = fu[s] * vp[min(4 * s + hi, c.cnt - 1) * in.v_stride];   // beta is 0 past cnt
    column(b, x, std::integral_constant<bool, false>{});
#pragma unroll
    for (int m = 0; m < 4; ++m) wu[(ct * 4 + m) * 64 + lane] = x[m];
  }
  f32x4* wk = (f32x4*)ws_k + (c.ws * heads + h) * (long)(4 * DKT * 64);
  for (int e = wave; e < 4 * DKT; e += 4) {
    const int i = e / 4, m = e % 4;
    f32x4 x;
#pragma unroll
    for (int r = 0; r < 4; ++r) x[r] = kb[(16 * m + 4 * hi + r) * LDK + 16 * i + lo] * el[16 * m + 4 * hi + r];
    wk[e * 64 + lane] = x;
  }
}

// ---------------------------------------------------------------------------------
// grid (heads, ceil(dv / 16), segments), four waves: the state's 16 columns, chunk after chunk.
// (Heads come first so that, 8 XCDs taking workgroups in turn, the column tiles of a head
// tend to share one XCD's L2: they all read the same operands.)
// Wave w holds the 16-row tiles w IT .. w IT + IT - 1 in accumulators; accumulator register r of
// lane (hi, lo) is row 4 hi + r, column lo, which is also a right-hand operand whose inner index
// 4 hi + r the left-hand operands (16-byte loads) follow.  Per chunk: every wave's part of
// -W S for all 64 rows, the parts added through LDS (wave w adds U and owns rows 16 w ..), w left
// in place of U, then S <- e^{G_last} S + K^T w.  Two register sets keep a chunk's operands
// on their way while the chunk before is computed.  FULL (whole tiles: dk = 16 DKT, dv a multiple of
// 16): no access is conditional, so nothing in the loop waits for more than it uses.
// ---------------------------------------------------------------------------------
template <int DKT, bool FULL>
__global__ void __launch_bounds__(256)
delta_carry_kernel(float* __restrict__ ws_s, const float* __restrict__ ws_w, const float* __restrict__ ws_k,
                   float* __restrict__ ws_u, const float* __restrict__ ws_g, float* __restrict__ state,
                   const int* __restrict__ start, const int* __restrict__ pos0, const int* __restrict__ slot, int heads,
                   int dk, int dv, int num_slots, int min_rows) {
  constexpr int IT = DKT < 4 ? 1 : DKT / 4;
  __shared__ f32x4 part[4][4][64], whole[4][64];
  Chunk c;
  if (!find_chunk(c, 0, blockIdx.z, start, pos0, slot, min_rows, num_slots)) return;
  const int h = blockIdx.x;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lo = lane & 15, hi = lane >> 4;
  const int col = blockIdx.y * 16 + lo;
  const bool live = FULL || col < dv;
  const bool mine = DKT >= 4 || wave * IT < DKT;     // few tiles: some waves only add
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
    idx = min(idx, c.num - 1);         // past the end: loaded again, not used
    const long cs = (c.ws + idx) * heads + h;
    const f32x4* w = (const f32x4*)ws_w + cs * (4 * DKT * 64) + lane;
    const f32x4* k = (const f32x4*)ws_k + cs * (4 * DKT * 64) + lane;
    if (mine) {
#pragma unroll
      for (int m = 0; m < 4; ++m)
#pragma unroll
        for (int ii = 0; ii < IT; ++ii) {
          const int i = wave * IT + ii;
          f.w[m][ii] = w[(m * DKT + i) * 64];
          f.k[ii][m] = k[(i * 4 + m) * 64];
        }
    }
    f.u = ((const f32x4*)ws_u)[((cs * gridDim.y + blockIdx.y) * 4 + wave) * 64 + lane];
    f.g = ws_g[cs];
    asm volatile("" ::: "memory");     // the loads stay here: they are not moved to their uses, two chunks on
  };
  auto turn = [&](const Ops& f, int idx) {
    float* so = ws_s + (((c.ws + idx) * heads + h) * dk) * (long)dv + col;
    if (mine && live) {
#pragma unroll
      for (int ii = 0; ii < IT; ++ii)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int row = 16 * (wave * IT + ii) + 4 * hi + r;
          if (FULL || row < dk) so[(long)row * dv] = S[ii][r];
        }
    }
    f32x4 a[4];
#pragma unroll
    for (int m = 0; m < 4; ++m) a[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (mine) {
#pragma unroll
      for (int ii = 0; ii < IT; ++ii)
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int m = 0; m < 4; ++m) a[m] = mma(f.w[m][ii][r], S[ii][r], a[m]);
    }
#pragma unroll
    for (int m = 0; m < 4; ++m) part[m][wave][lane] = a[m];
    __syncthreads();
    {
      const f32x4 v0 = part[wave][0][lane], v1 = part[wave][1][lane], v2 = part[wave][2][lane], v3 = part[wave][3][lane];
      a[0] = (f.u + v0) + (v1 + (v2 + v3));
    }
    const f32x4 v = a[0];
    whole[wave][lane] = v;
    ((f32x4*)ws_u)[((((c.ws + idx) * heads + h) * gridDim.y + blockIdx.y) * 4 + wave) * 64 + lane] = v;
    __syncthreads();
    if (mine) {
      f32x4 vm[4], e[IT][2];             // two sums per tile in turn
#pragma unroll
      for (int m = 0; m < 4; ++m) vm[m] = whole[m][lane];
#pragma unroll
      for (int ii = 0; ii < IT; ++ii) {
        e[ii][0] = S[ii] * f.g;
        e[ii][1] = f32x4{0.f, 0.f, 0.f, 0.f};
      }
#pragma unroll
      for (int m = 0; m < 4; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int ii = 0; ii < IT; ++ii) e[ii][r & 1] = mma(f.k[ii][m][r], vm[m][r], e[ii][r & 1]);
#pragma unroll
      for (int ii = 0; ii < IT; ++ii) S[ii] = e[ii][0] + e[ii][1];
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
  const int vec = dk % 4 == 0 && dv % 4 == 0 && (((uintptr_t)q | (uintptr_t)k | (uintptr_t)v) % 16) == 0;
  if (((uintptr_t)ws_w | (uintptr_t)ws_k | (uintptr_t)ws_u) % 16) return -3;
  const int chunks = (max_rows + kC - 1) / kC;
  if (heads > 65535 || (long)heads * ((dv + 63) / 64) > 65535 || num_segs > 65535) return -2;
  key_tiles(dk, [&](auto t) {
    hipLaunchKernelGGL((delta_solve_kernel<decltype(t)::value>), dim3(chunks, heads, num_segs), dim3(256), 0, s, ws_w,
                       ws_k, ws_u, ws_g, in, beta, start, pos0, slot, heads, dk, dv, num_slots, min_rows, vec);
    constexpr int DKT = decltype(t)::value;
    const dim3 cgrid(heads, (dv + 15) / 16, num_segs);
    if (dk == 16 * DKT && dv % 16 == 0)
      hipLaunchKernelGGL((delta_carry_kernel<DKT, true>), cgrid, dim3(256), 0, s, ws_s, ws_w, ws_k, ws_u, ws_g, state, start,
                         pos0, slot, heads, dk, dv, num_slots, min_rows);
    else
      hipLaunchKernelGGL((delta_carry_kernel<DKT, false>), cgrid, dim3(256), 0, s, ws_s, ws_w, ws_k, ws_u, ws_g, state, start,
                         pos0, slot, heads, dk, dv, num_slots, min_rows);
  });
  in.v = ws_u;                     // the solved rows take the values' place
  in.v_frags = 1;
  launch_out<float>(o, in, ws_s, start, pos0, slot, dim3(chunks, heads * ((dv + 63) / 64), num_segs), heads, dk, dv,
                    num_slots, min_rows, vec, s);
  return (int)hipGetLastError();
}
