// Recurrences with one decay per head over fp32 state slots, walked row by row (decode rows
// and short segments): the gated delta rule and retention; and the preparation of the delta
// rule's inputs.  Long segments take the chunk form in chunk_state.hip.
//
// Rows come in segments as in delta_rule.hip (start / pos0 / slot; a segment at position 0
// starts from zeros; slot < 0 is padding).  Per head, S [dk, dv] fp32:
//   delta rule:  S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//   retention:   S <- d S + k v^T;  o = S^T q           (d fixed per head)
// q and k of the delta rule come prepared (conv_delta_prep_kernel); retention reads the raw
// projection and rotates q and k by position while staging them.
//
// Columns of S are independent: a workgroup of 256 threads owns 32 columns of one head of one
// sequence, 8 lanes of 4 neighbouring columns each (16-byte accesses of the state) times 32
// row groups (rows rg, rg + 32, ...), so a single decode row reads and writes its share of the
// state in one sweep with every load in flight.  For the delta rule both dot products of a
// row are taken of the state before the row, S_old^T k and S_old^T q, and reduced together;
// the read-out after the write is then g S_old^T q + (k.q) u.
#include "mx_common.h"

namespace mx {

constexpr int kHCols = 32;      // state columns per workgroup
constexpr int kHRows = 8;       // rows staged at a time

// v plus the v of the lane 8 away within a row of 16
__device__ __forceinline__ float add_eights(float v) {
  return v + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x128, 0xF, 0xF, true));
}
// sum over the lanes 8, 16 and 32 away: the 8 lanes of a wave that share lane % 8
__device__ __forceinline__ float sum_groups8(float v) { return add_halves(add_row_pair(add_eights(v))); }

struct HeadIn {
  const void* q;              // delta: fp32 [T, kv_heads, dk]; retention: the projection's rows (T)
  const void* k;
  const void* v;
  long q_stride, k_stride, v_stride;   // elements between rows
  int rep;                    // heads per q / k head
  const float* lg;            // delta: log decay [T, heads]
  const float* beta;          // delta: [T, heads]
  const double* log_decay;    // retention: [heads]
  const float* table;         // retention: [cos | sin] rows, null: no rotation
  int table_rows, rot_dims, interleaved;
  float k_scale;              // retention
};

template <typename T, bool DELTA, int R>
__global__ void __launch_bounds__(256)
head_walk_kernel(float* __restrict__ o, HeadIn in, float* __restrict__ state, const int* __restrict__ start,
                 const int* __restrict__ pos0, const int* __restrict__ slot, int heads, int dk, int dv, int num_slots,
                 int skip_from, int vec) {
  constexpr int NP = 32 * R;
  __shared__ float k_s[kHRows][NP], q_s[kHRows][NP];
  __shared__ __attribute__((aligned(16))) float v_s[kHRows][kHCols];
  __shared__ float g_s[kHRows], b_s[kHRows];
  // delta: per parity, wave and column group the sums [S^T k | S^T q] of 4 columns, and k.q;
  // retention: per row and wave the outputs of the 32 columns
  __shared__ __attribute__((aligned(16))) float red[DELTA ? 2 : kHRows][4][DELTA ? 72 : kHCols];
  const int s = blockIdx.z, h = blockIdx.y;
  const int r0 = start[s], n = start[s + 1] - r0;
  if (n <= 0 || (skip_from > 0 && n >= skip_from)) return;
  const int sl = slot[s];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int cg = tid & 7, rg = tid >> 3;
  const int tile0 = blockIdx.x * kHCols, col = tile0 + 4 * cg;
  const long o_stride = (long)heads * dv;
  float* op = o + (long)r0 * o_stride + (long)h * dv;
  if (sl < 0 || sl >= num_slots) {
    for (int e = tid; e < n * kHCols; e += 256)
      if (tile0 + e % kHCols < dv) op[(long)(e / kHCols) * o_stride + tile0 + e % kHCols] = 0.f;
    return;
  }
  float* S = state + (((long)sl * heads + h) * dk) * dv;
  const bool fresh = pos0[s] <= 0;
  float st_[R][4];
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int r = rg + 32 * i;
    if (fresh || r >= dk || col >= dv) {
#pragma unroll
      for (int c = 0; c < 4; ++c) st_[i][c] = 0.f;
    } else if (vec) {
      const float4 u = *reinterpret_cast<const float4*>(S + (long)r * dv + col);
      st_[i][0] = u.x; st_[i][1] = u.y; st_[i][2] = u.z; st_[i][3] = u.w;
    } else {
#pragma unroll
      for (int c = 0; c < 4; ++c) st_[i][c] = col + c < dv ? S[(long)r * dv + col + c] : 0.f;
    }
  }
  const long qoff = (long)(h / in.rep) * dk, voff = (long)h * dv + tile0;
  float decay = 1.f;
  if constexpr (!DELTA) decay = (float)exp(in.log_decay[h]);

  for (int t0 = 0; t0 < n; t0 += kHRows) {
    const int cnt = min(kHRows, n - t0);
    for (int e = tid; e < cnt * NP; e += 256) {
      const int t = e / NP, i = e % NP;
      const long row = r0 + t0 + t;
      float kv = 0.f, qv = 0.f;
      if (i < dk) {
        const T* qp = (const T*)in.q + row * in.q_stride + qoff;
        const T* kp = (const T*)in.k + row * in.k_stride + qoff;
        if (!DELTA && in.table != nullptr && i < in.rot_dims) {
          int pos = pos0[s] + t0 + t;
          if (pos < 0 || pos >= in.table_rows) pos = 0;
          const float* cs = in.table + (long)pos * in.rot_dims;
          qv = rope_at(qp, i, in.rot_dims, cs, in.interleaved);
          kv = rope_at(kp, i, in.rot_dims, cs, in.interleaved);
        } else {
          qv = ld(qp, i);
          kv = ld(kp, i);
        }
        if constexpr (!DELTA) kv *= in.k_scale;
      }
      q_s[t][i] = qv;
      k_s[t][i] = kv;
    }
    for (int e = tid; e < cnt * kHCols; e += 256) {
      const int t = e / kHCols, c = e % kHCols;
      v_s[t][c] = tile0 + c < dv ? ld((const T*)in.v, (long)(r0 + t0 + t) * in.v_stride + voff + c) : 0.f;
    }
    if constexpr (DELTA) {
      if (tid < cnt) {
        g_s[tid] = expf(in.lg[(long)(r0 + t0 + tid) * heads + h]);
        b_s[tid] = in.beta[(long)(r0 + t0 + tid) * heads + h];
      }
    }
    __syncthreads();
    for (int t = 0; t < cnt; ++t) {
      float kk[R], qq[R];
#pragma unroll
      for (int i = 0; i < R; ++i) {
        kk[i] = k_s[t][rg + 32 * i];
        qq[i] = q_s[t][rg + 32 * i];
      }
      const float4 v4 = *reinterpret_cast<const float4*>(&v_s[t][4 * cg]);
      const float vv[4] = {v4.x, v4.y, v4.z, v4.w};
      if constexpr (DELTA) {
        float pk[4] = {0.f, 0.f, 0.f, 0.f}, pq[4] = {0.f, 0.f, 0.f, 0.f}, kq = 0.f;
#pragma unroll
        for (int i = 0; i < R; ++i) {
          kq += kk[i] * qq[i];
#pragma unroll
          for (int c = 0; c < 4; ++c) {
            pk[c] += st_[i][c] * kk[i];
            pq[c] += st_[i][c] * qq[i];
          }
        }
        kq = sum_groups8(kq);
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          pk[c] = sum_groups8(pk[c]);
          pq[c] = sum_groups8(pq[c]);
        }
        float(*rd)[72] = red[t & 1];
        if (lane < 8) {
#pragma unroll
          for (int c = 0; c < 4; ++c) {
            rd[wave][4 * lane + c] = pk[c];
            rd[wave][32 + 4 * lane + c] = pq[c];
          }
          if (lane == 0) rd[wave][64] = kq;
        }
        __syncthreads();
        const float g = g_s[t], b = b_s[t];
        float u[4];
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          const float dot = (rd[0][4 * cg + c] + rd[1][4 * cg + c]) + (rd[2][4 * cg + c] + rd[3][4 * cg + c]);
          u[c] = b * (vv[c] - g * dot);
        }
#pragma unroll
        for (int i = 0; i < R; ++i)
#pragma unroll
          for (int c = 0; c < 4; ++c) st_[i][c] = g * st_[i][c] + kk[i] * u[c];
        if (tid < 8) {
          const float kqs = (rd[0][64] + rd[1][64]) + (rd[2][64] + rd[3][64]);
#pragma unroll
          for (int c = 0; c < 4; ++c) {
            const int x = 32 + 4 * cg + c;
            const float out = g * ((rd[0][x] + rd[1][x]) + (rd[2][x] + rd[3][x])) + kqs * u[c];
            if (col + c < dv) op[(long)(t0 + t) * o_stride + col + c] = out;
          }
        }
      } else {
        float pq[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < R; ++i)
#pragma unroll
          for (int c = 0; c < 4; ++c) {
            st_[i][c] = decay * st_[i][c] + kk[i] * vv[c];
            pq[c] += st_[i][c] * qq[i];
          }
#pragma unroll
        for (int c = 0; c < 4; ++c) pq[c] = sum_groups8(pq[c]);
        if (lane < 8)
          *reinterpret_cast<float4*>(&red[t][wave][4 * lane]) = make_float4(pq[0], pq[1], pq[2], pq[3]);
      }
    }
    __syncthreads();          // the staged rows (and retention's outputs of them) are complete / free
    if constexpr (!DELTA) {
      for (int e = tid; e < cnt * kHCols; e += 256) {
        const int t = e / kHCols, c = e % kHCols;
        if (tile0 + c < dv)
          op[(long)(t0 + t) * o_stride + tile0 + c] = (red[t][0][c] + red[t][1][c]) + (red[t][2][c] + red[t][3][c]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int r = rg + 32 * i;
    if (r >= dk || col >= dv) continue;
    if (vec) {
      *reinterpret_cast<float4*>(S + (long)r * dv + col) = make_float4(st_[i][0], st_[i][1], st_[i][2], st_[i][3]);
    } else {
#pragma unroll
      for (int c = 0; c < 4; ++c)
        if (col + c < dv) S[(long)r * dv + col + c] = st_[i][c];
    }
  }
}

// ---------------------------------------------------------------------------------
// inputs of the delta rule with one decay per head, one wave per (RB rows, item): items are the
// 2 kv_heads heads of q and k, then v in pieces of 64 NU channels, then one item for all heads'
// decays and steps.  Every channel of q, k and v passes its causal convolution over time (rows
// before the segment's first come from the slot's history, zeros at position 0) and silu, in
// fp32; a q or k head is then divided by its length.  A one-row segment leaves its history here
// (each channel is one lane's own); longer ones are left to conv_hist_kernel.
// ---------------------------------------------------------------------------------
template <typename T, int TAPS, int NU, int RB>
__global__ void __launch_bounds__(256)
conv_delta_prep_kernel(float* __restrict__ qn, float* __restrict__ kn, float* __restrict__ vo, float* __restrict__ lg,
                       float* __restrict__ beta, const T* __restrict__ x, long x_stride, const T* __restrict__ a,
                       long a_stride, const T* __restrict__ b, long b_stride, const float* __restrict__ conv_w,
                       int taps, float* hist, const float* __restrict__ a_log, const float* __restrict__ dt_bias,
                       const int* __restrict__ start, const int* __restrict__ pos0, const int* __restrict__ slot,
                       int num_segs, int num_slots, int heads, int kv_heads, int dk, int dv) {
  const int lane = threadIdx.x & 63;
  const int item = blockIdx.y * 4 + (threadIdx.x >> 6);
  const int row0 = blockIdx.x * RB, rows = start[num_segs];
  const int qk = 2 * kv_heads, nv = heads * dv, pieces = (nv + 64 * NU - 1) / (64 * NU);
  if (item > qk + pieces || row0 >= rows) return;
  if (item == qk + pieces) {
    for (int e = lane; e < RB * heads; e += 64) {
      const int row = row0 + e / heads, h = e % heads;
      if (row >= rows) break;
      const float z = ld(a, (long)row * a_stride + h) + dt_bias[h];
      lg[(long)row * heads + h] = -expf(a_log[h]) * softplusf_(z);
      beta[(long)row * heads + h] = sigmoidf_(ld(b, (long)row * b_stride + h));
    }
    return;
  }
  const bool is_v = item >= qk, is_q = item < kv_heads;
  const int channels = qk * dk + nv;
  const int c0 = is_v ? qk * dk + (item - qk) * 64 * NU : item * dk;
  const int len = is_v ? min(64 * NU, channels - c0) : dk;
  float xs[RB][NU];
#pragma unroll
  for (int r = 0; r < RB; ++r)
#pragma unroll
    for (int u = 0; u < NU; ++u) {
      const int i = lane + 64 * u;
      xs[r][u] = ld(x, (long)min(row0 + r, rows - 1) * x_stride + c0 + (i < len ? i : 0));
    }
  ConvWalk<TAPS, NU> cv;
  cv.weights(conv_w, taps, c0, len, lane);
  int s = segment_of(start, num_segs, row0), at = -1;
  const float qscale = is_q ? 1.0f / sqrtf((float)dk) : 1.f;
#pragma unroll
  for (int r = 0; r < RB; ++r) {
    const int row = row0 + r;
    if (row >= rows) break;
    while (row >= start[s + 1]) ++s;
    float* h = nullptr;
    if (s != at) {
      const int sl = slot[s];
      const bool mine = sl >= 0 && sl < num_slots;
      if (mine) h = hist + (long)sl * (taps - 1) * channels;
      cv.begin(x, x_stride, start[s], row - start[s], mine && pos0[s] > 0 ? h : nullptr, channels, taps, c0, len, lane);
      at = s;
    }
    float y[NU], ss = 0.f;
#pragma unroll
    for (int u = 0; u < NU; ++u) {
      const float z = cv.step(u, xs[r][u]);
      cv.shift(u);
      y[u] = lane + 64 * u < len ? z * sigmoidf_(z) : 0.f;
      ss += y[u] * y[u];
    }
    if (h != nullptr && start[s + 1] - start[s] == 1) cv.store(h, channels, taps, c0, len, lane);
    float* out;
    float f = 1.f;
    if (is_v) {
      out = vo + (long)row * nv + (item - qk) * 64 * NU;
    } else {
      out = (is_q ? qn : kn) + ((long)row * kv_heads + (is_q ? item : item - kv_heads)) * dk;
      f = 1.0f / sqrtf(ft::wave_sum(ss) + 1e-6f) * qscale;
    }
#pragma unroll
    for (int u = 0; u < NU; ++u)
      if (lane + 64 * u < len) out[lane + 64 * u] = y[u] * f;
  }
}

}  // namespace mx

using namespace mx;

extern "C" int mx_conv_hist(const void* x, int bf16, long x_stride, float* hist, const int* start, const int* pos0,
                            const int* slot, int num_segs, int channels, int taps, int num_slots, int min_rows,
                            hipStream_t s);

extern "C" int mx_head_max_dk() { return 256; }

extern "C" int mx_conv_delta_prep(float* qn, float* kn, float* vo, float* lg, float* beta, const void* x, int bf16,
                                  long x_stride, const void* a, long a_stride, const void* b, long b_stride,
                                  const float* conv_w, int taps, float* hist, const float* a_log, const float* dt_bias,
                                  const int* start, const int* pos0, const int* slot, int num_segs, int max_rows,
                                  long rows, int num_slots, int heads, int kv_heads, int dk, int dv, hipStream_t s) {
  if (rows <= 0 || num_segs <= 0) return 0;
  if (taps < 1 || taps > 16 || dk < 1 || dk > mx_head_max_dk() || dv < 1 || kv_heads < 1 || heads % kv_heads) return -1;
  // rows per wave: a few once there are enough of them
  const int rb = rows >= 256 ? 8 : 1, nu = dk <= 64 ? 1 : dk <= 128 ? 2 : 4;
  const int items = 2 * kv_heads + (heads * dv + 64 * nu - 1) / (64 * nu) + 1;
  if (rows > 0x7fffffffL || (items + 3) / 4 > 65535) return -2;
  const dim3 grid((unsigned)((rows + rb - 1) / rb), (unsigned)((items + 3) / 4));
#define MX_CDP(TAPS, NU, RB)                                                                                      \
  MX_DISPATCH_T(bf16, hipLaunchKernelGGL((conv_delta_prep_kernel<T, TAPS, NU, RB>), grid, dim3(256), 0, s, qn, kn, vo, \
                                         lg, beta, (const T*)x, x_stride, (const T*)a, a_stride, (const T*)b, b_stride, \
                                         conv_w, taps, hist, a_log, dt_bias, start, pos0, slot, num_segs, num_slots,  \
                                         heads, kv_heads, dk, dv))
#define MX_CDN(TAPS, RB)            \
  do {                              \
    if (nu == 1) MX_CDP(TAPS, 1, RB); \
    else if (nu == 2) MX_CDP(TAPS, 2, RB); \
    else MX_CDP(TAPS, 4, RB);       \
  } while (0)
  if (taps <= 4 && rb == 8) MX_CDN(4, 8);
  else if (taps <= 4) MX_CDN(4, 1);
  else if (rb == 8) MX_CDN(16, 8);
  else MX_CDN(16, 1);
#undef MX_CDN
#undef MX_CDP
  int rc = (int)hipGetLastError();
  if (rc == 0 && taps > 1 && max_rows > 1)
    rc = mx_conv_hist(x, bf16, x_stride, hist, start, pos0, slot, num_segs, 2 * kv_heads * dk + heads * dv, taps,
                      num_slots, 2, s);
  return rc;
}

template <typename T, bool DELTA>
static int launch_walk(float* o, const HeadIn& in, float* state, const int* start, const int* pos0, const int* slot,
                       int num_segs, int heads, int dk, int dv, int num_slots, int skip_from, hipStream_t s) {
  const dim3 grid((dv + kHCols - 1) / kHCols, heads, num_segs);
  if (grid.y > 65535 || grid.z > 65535) return -2;
  const int vec = dv % 4 == 0 && ((uintptr_t)state) % 16 == 0;
  const int need = (dk + 31) / 32;
#define MX_WALK(R)                                                                                              \
  hipLaunchKernelGGL((head_walk_kernel<T, DELTA, R>), grid, dim3(256), 0, s, o, in, state, start, pos0, slot, heads, \
                     dk, dv, num_slots, skip_from, vec)
  if (need <= 1) MX_WALK(1);
  else if (need <= 2) MX_WALK(2);
  else if (need <= 4) MX_WALK(4);
  else MX_WALK(8);
#undef MX_WALK
  return (int)hipGetLastError();
}

extern "C" int mx_head_delta_walk(float* o, const float* q, const float* k, const float* v, const float* lg,
                                  const float* beta, float* state, const int* start, const int* pos0, const int* slot,
                                  int num_segs, int heads, int kv_heads, int dk, int dv, int num_slots, int skip_from,
                                  hipStream_t s) {
  if (num_segs <= 0) return 0;
  if (dk < 1 || dk > mx_head_max_dk() || dv < 1 || kv_heads < 1 || heads % kv_heads) return -1;
  HeadIn in{};
  in.q = q; in.k = k; in.v = v;
  in.q_stride = in.k_stride = (long)kv_heads * dk;
  in.v_stride = (long)heads * dv;
  in.rep = heads / kv_heads;
  in.lg = lg; in.beta = beta;
  return launch_walk<float, true>(o, in, state, start, pos0, slot, num_segs, heads, dk, dv, num_slots, skip_from, s);
}

extern "C" int mx_retention_walk(float* o, const void* p, int bf16, long stride, const float* table, int table_rows,
                                 int rot_dims, int interleaved, const double* log_decay, float* state,
                                 const int* start, const int* pos0, const int* slot, int num_segs, int heads, int dk,
                                 int dv, int num_slots, int skip_from, hipStream_t s) {
  if (num_segs <= 0) return 0;
  if (dk < 1 || dk > mx_head_max_dk() || dv < 1 || heads < 1) return -1;
  HeadIn in{};
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
  int rc = 0;
  MX_DISPATCH_T(bf16, rc = (launch_walk<T, false>(o, in, state, start, pos0, slot, num_segs, heads, dk, dv, num_slots,
                                                  skip_from, s)));
  return rc;
}
