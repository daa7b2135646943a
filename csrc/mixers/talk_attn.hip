// Grouped-query attention that mixes its scores across the heads before the softmax, over a
// paged key cache and a paged value cache.
//
// Query head h reads key and value head h / rep, rep = heads / kv_heads.  Position i sees
// key j iff j <= i and (i - j < window, or window == 0, or j < keep_first).  With dot
// products s_g = q_g . k (queries come scaled): s_g <- softcap tanh(s_g / softcap) when
// softcap > 0, z_h = sum_g talk[h][g] s_g, weights = softmax of z_h over the visible keys.
// Every head's weight of a key needs all heads' scores of that key, so the unit of work is
// a tile of keys for all heads together.
// Queries, scores, weights and sums are fp32; the caches hold fp32 or bf16 rows.
//
// Kernels: rot_norm_prep (rotary positions, per-head RMS norms, cache writes),
// talk_attn + talk_combine (decode rows and short segments: key slices of a row, merged,
// gated and rounded), talk_weights (scores -> weights for the banded matrix products of
// long segments) and heads_to_rows (per-head results -> gated rows).
#include "mx_common.h"

namespace mx {

// ---------------------------------------------------------------------------------
// one wave per (row, head) of the q and k parts of a fused projection: rotary positions on
// the head's first rot_dims entries, then the head divided by its root mean square.  q
// leaves as fp32 times q_scale[head]; k goes to the row's key slot, and as projected
// (before rotation and norm) to its value slot.  grid (rows, ceil(heads / 4)), 4 waves.
// ---------------------------------------------------------------------------------
constexpr int kPrepCols = 8;      // entries per lane: head_dim <= 512

template <typename T, typename TC>
__global__ void __launch_bounds__(256)
rot_norm_prep_kernel(float* __restrict__ q_out, const T* __restrict__ qk, long stride, int q_heads, int k_heads,
                     int head_dim, const float* __restrict__ table, int table_rows, int rot_dims, int interleaved,
                     float eps, const float* __restrict__ q_scale, const int* __restrict__ positions,
                     const int* __restrict__ slots, TC* __restrict__ k_cache, TC* __restrict__ v_cache,
                     long num_slots) {
  const int lane = threadIdx.x & 63;
  const int hd = blockIdx.y * 4 + (threadIdx.x >> 6);
  const long row = blockIdx.x;
  if (hd >= q_heads + k_heads) return;
  int pos = positions[row];
  if (pos < 0 || pos >= table_rows) pos = 0;
  const float* cs = table + (long)pos * rot_dims;      // not read when rot_dims == 0
  const T* x = qk + row * stride + (long)hd * head_dim;
  float y[kPrepCols], raw[kPrepCols];
  float ss = 0.f;
#pragma unroll
  for (int u = 0; u < kPrepCols; ++u) {
    const int d = lane + 64 * u;
    y[u] = raw[u] = 0.f;
    if (d < head_dim) {
      raw[u] = ld(x, d);
      y[u] = d < rot_dims ? rope_at(x, d, rot_dims, cs, interleaved) : raw[u];
      ss += y[u] * y[u];
    }
  }
  const float r = 1.0f / sqrtf(ft::wave_sum(ss) / (float)head_dim + eps);
  if (hd < q_heads) {
    const float f = r * q_scale[hd];
    float* qp = q_out + (row * q_heads + hd) * head_dim;
#pragma unroll
    for (int u = 0; u < kPrepCols; ++u) {
      const int d = lane + 64 * u;
      if (d < head_dim) qp[d] = y[u] * f;
    }
    return;
  }
  const long slot = slots[row];
  if (slot < 0 || slot >= num_slots) return;
  const long base = (slot * k_heads + (hd - q_heads)) * head_dim;
#pragma unroll
  for (int u = 0; u < kPrepCols; ++u) {
    const int d = lane + 64 * u;
    if (d < head_dim) {
      st(k_cache, base + d, y[u] * r);
      st(v_cache, base + d, raw[u]);
    }
  }
}

// ---------------------------------------------------------------------------------
// decode rows and short segments: one workgroup of four waves per (row, slice of its
// keys), 64 keys per tile.
//   scores: lane = key; a wave takes groups of HU query heads that share a key head, so a
//           key row is read once per group (16-byte pieces against the queries in LDS);
//           the capped scores of all heads meet in LDS
//   mix + softmax: a wave owns HPW consecutive heads, lane = key
//   sums:   a lane owns one 16-byte piece of the value row of every (64 / LPK)-th key, as in
//           window_attn_kernel, for all of the wave's heads at once (VEC), or lane = column
// Each slice leaves (max, sum, weighted sums) per head for talk_combine_kernel.
// ---------------------------------------------------------------------------------
constexpr int kTalkWaves = 4;
constexpr int kTalkTile = 64;

template <typename TC> struct Row16;
template <> struct Row16<float> {
  static constexpr int N = 4;
  static __device__ __forceinline__ void load(const float* p, float* v) {
    const float4 u = *reinterpret_cast<const float4*>(p);
    v[0] = u.x; v[1] = u.y; v[2] = u.z; v[3] = u.w;
  }
};
template <> struct Row16<bf16_t> {
  static constexpr int N = 8;
  static __device__ __forceinline__ void load(const bf16_t* p, float* v) {
    const uint4 u = *reinterpret_cast<const uint4*>(p);
    const uint32_t w[4] = {u.x, u.y, u.z, u.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      v[2 * i] = __uint_as_float(w[i] << 16);
      v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
  }
};

// the visible keys of a row: key index c maps to position c < ext ? c : first + c - ext
struct TalkBand {
  int i, first, ext, nkeys;
};

__device__ __forceinline__ TalkBand talk_band(int i, int kv_len, int window, int keep_first) {
  TalkBand b;
  b.i = i;
  const int last = min(i, kv_len - 1);        // padding rows (empty context) see nothing
  b.first = window > 0 ? max(0, i - window + 1) : 0;
  b.ext = window > 0 ? max(0, min(min(keep_first, b.first), last + 1)) : 0;
  b.nkeys = b.ext + max(0, last - b.first + 1);
  return b;
}

constexpr int kScalarCols = 8;                // value columns per lane (scalar form): dv <= 512

template <typename TC, int HPW, int HU, bool VEC>
__global__ void __launch_bounds__(64 * kTalkWaves)
talk_attn_kernel(float* __restrict__ ws_acc, float* __restrict__ ws_ml, const float* __restrict__ q,
                 const TC* __restrict__ k_cache, const TC* __restrict__ v_cache, const int* __restrict__ start,
                 const int* __restrict__ pos0, const int* __restrict__ kv_len, const int* __restrict__ bt,
                 int bt_stride, int num_segs, int heads, int kv_heads, int dk, int dv, int window, int keep_first,
                 float softcap, const float* __restrict__ talk, int block_size, int num_blocks, int skip_from,
                 int splits, int vec, int lpk) {
  extern __shared__ float smem[];
  const long row = blockIdx.x / splits;
  const int sp = blockIdx.x % splits;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  if (row >= start[num_segs]) return;
  int lo_s = 0, hi_s = num_segs;
  while (hi_s - lo_s > 1) {
    const int mid = (lo_s + hi_s) >> 1;
    if (start[mid] <= row) lo_s = mid; else hi_s = mid;
  }
  const int s = lo_s;
  const int r0 = start[s], n = start[s + 1] - r0;
  if (skip_from > 0 && n >= skip_from) return;
  float* q_s = smem;                                 // [heads][dk]
  float* s_s = q_s + (long)heads * dk;               // [heads][64] capped scores
  float* p_s = s_s + heads * kTalkTile;              // [heads][64] weights
  const float* qp = q + row * (long)heads * dk;
  for (int d = tid; d < heads * dk; d += 64 * kTalkWaves) q_s[d] = qp[d];
  const int rep = heads / kv_heads;
  const long nk = (long)kv_heads * dk, nv = (long)kv_heads * dv;
  const TalkBand b = talk_band(pos0[s] + (int)(row - r0), kv_len[s], window, keep_first);
  const int tiles = (b.nkeys + kTalkTile - 1) / kTalkTile;
  const int per = (tiles + splits - 1) / splits * kTalkTile;
  const int begin = min(sp * per, b.nkeys), end = min(begin + per, b.nkeys);
  const int* table = bt + (long)s * bt_stride;
  const int h0 = wave * HPW;                         // this wave's heads h0 .. h0 + HPW - 1 (< heads)
  const int upg = (rep + HU - 1) / HU, units = kv_heads * upg;

  constexpr int NO = VEC ? Row16<TC>::N : kScalarCols;
  float o[HPW][NO], m[HPW], l[HPW];
#pragma unroll
  for (int x = 0; x < HPW; ++x) {
    m[x] = -INFINITY;
    l[x] = 0.f;
#pragma unroll
    for (int u = 0; u < NO; ++u) o[x][u] = 0.f;
  }
  const int pieces = dv / Row16<TC>::N;
  const int sg = lane & (lpk - 1), sub = lane / lpk, kpp = 64 / lpk;
  const bool has_piece = sg < pieces;
  for (int c0 = begin; c0 < end; c0 += kTalkTile) {
    const int cc = c0 + lane;
    const int j = cc < b.ext ? cc : b.first + cc - b.ext;
    int slot = -1;
    if (cc < end) {
      const int blk = table[j / block_size];
      if (blk >= 0 && blk < num_blocks) slot = blk * block_size + j % block_size;
    }
    __syncthreads();                                 // q_s is there / the last tile's s_s is no longer read
    const TC* krow = k_cache + (long)max(slot, 0) * nk;
    for (int u = wave; u < units; u += kTalkWaves) {
      const int g = u / upg, x0 = (u % upg) * HU, hb = g * rep + x0;
      const int nh = min(HU, rep - x0);
      const TC* kp = krow + (long)g * dk;
      float acc[HU];
#pragma unroll
      for (int x = 0; x < HU; ++x) acc[x] = 0.f;
      const float* qh[HU];
#pragma unroll
      for (int x = 0; x < HU; ++x) qh[x] = q_s + (long)(hb + min(x, nh - 1)) * dk;
      if (vec) {
        constexpr int N = Row16<TC>::N;
#pragma unroll 4
        for (int d = 0; d < dk; d += N) {
          float kv[N];
          Row16<TC>::load(kp + d, kv);
#pragma unroll
          for (int x = 0; x < HU; ++x)
#pragma unroll
            for (int e = 0; e < N; e += 4) {
              const float4 q4 = *reinterpret_cast<const float4*>(qh[x] + d + e);
              acc[x] += q4.x * kv[e] + q4.y * kv[e + 1] + q4.z * kv[e + 2] + q4.w * kv[e + 3];
            }
        }
      } else {
        for (int d = 0; d < dk; ++d) {
          const float kv = ld(kp, d);
#pragma unroll
          for (int x = 0; x < HU; ++x) acc[x] += qh[x][d] * kv;
        }
      }
#pragma unroll
      for (int x = 0; x < HU; ++x)
        if (x < nh) {
          float z = acc[x];
          if (softcap > 0.f) z = softcap * tanhf(z / softcap);
          s_s[(hb + x) * kTalkTile + lane] = z;
        }
    }
    __syncthreads();
    if (h0 < heads) {
#pragma unroll
      for (int x = 0; x < HPW; ++x) {
        const int h = h0 + x;
        if (h >= heads) break;
        const float* tr = talk + (long)h * heads;
        float z = 0.f;
        for (int g = 0; g < heads; ++g) z += tr[g] * s_s[g * kTalkTile + lane];
        if (slot < 0) z = -INFINITY;
        const float mn = fmaxf(m[x], ft::wave_max(z));
        const float resc = m[x] == -INFINITY ? 0.f : expf(m[x] - mn);
        const float p = (slot >= 0 && mn != -INFINITY) ? expf(z - mn) : 0.f;
        l[x] = l[x] * resc + ft::wave_sum(p);
        m[x] = mn;
        p_s[h * kTalkTile + lane] = p;
#pragma unroll
        for (int u = 0; u < NO; ++u) o[x][u] *= resc;
      }
      // the wave's own LDS writes, read by its other lanes
      __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
      const int cnt = min(kTalkTile, end - c0);
      if constexpr (VEC) {
        const int passes = (cnt + kpp - 1) / kpp;
#pragma unroll 4
        for (int ps = 0; ps < passes; ++ps) {
          const int jj = ps * kpp + sub;             // < 64: a key past cnt has weight 0, slot -1
          const int sj = __shfl(slot, jj);
          const bool ok = sj >= 0 && has_piece;
          const TC* vrow = v_cache + (ok ? (long)sj * nv + sg * Row16<TC>::N : 0L);
          float v[Row16<TC>::N];
#pragma unroll
          for (int x = 0; x < HPW; ++x) {
            const int h = min(h0 + x, heads - 1), g = h / rep;
            if (x == 0 || g != min(h0 + x - 1, heads - 1) / rep) Row16<TC>::load(vrow + (ok ? (long)g * dv : 0L), v);
            const float w = ok ? p_s[h * kTalkTile + jj] : 0.f;
#pragma unroll
            for (int u = 0; u < Row16<TC>::N; ++u) o[x][u] += w * v[u];
          }
        }
      } else {
        for (int jj = 0; jj < cnt; ++jj) {
          const int sj = __shfl(slot, jj);
          if (sj < 0) continue;
#pragma unroll
          for (int x = 0; x < HPW; ++x) {
            const int h = min(h0 + x, heads - 1);
            const TC* vp = v_cache + (long)sj * nv + (long)(h / rep) * dv;
            const float w = p_s[h * kTalkTile + jj];
#pragma unroll
            for (int u = 0; u < kScalarCols; ++u) {
              const int c = lane + 64 * u;
              if (c < dv) o[x][u] += w * ld(vp, c);
            }
          }
        }
      }
    }
  }
  const long base = (row * splits + sp) * heads;
#pragma unroll
  for (int x = 0; x < HPW; ++x) {
    const int h = h0 + x;
    if (h >= heads) break;
    float* dst = ws_acc + (base + h) * dv;
    if constexpr (VEC) {
      // lanes sub = 0, 1, ... hold partial sums of the same piece
      for (int off = lpk; off < 64; off <<= 1) {
#pragma unroll
        for (int u = 0; u < NO; ++u) o[x][u] += __shfl_xor(o[x][u], off);
      }
      if (sub == 0 && has_piece) {
#pragma unroll
        for (int u = 0; u < NO; ++u) dst[sg * Row16<TC>::N + u] = o[x][u];
      }
    } else {
#pragma unroll
      for (int u = 0; u < kScalarCols; ++u) {
        const int c = lane + 64 * u;
        if (c < dv) dst[c] = o[x][u];
      }
    }
    if (lane == 0) {
      ws_ml[(base + h) * 2] = m[x];
      ws_ml[(base + h) * 2 + 1] = l[x];
    }
  }
}

// one wave per (row, head): merges the slices, divides by the sum, applies the element-wise
// sigmoid gate (optional) and rounds
template <typename TG, typename TO>
__global__ void __launch_bounds__(256)
talk_combine_kernel(TO* __restrict__ out, const float* __restrict__ ws_acc, const float* __restrict__ ws_ml,
                    const TG* __restrict__ gate, long gate_stride, const int* __restrict__ start, int num_segs,
                    long total_rows, int heads, int dv, int skip_from, int splits) {
  const long pair = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (pair >= total_rows * heads) return;
  const int lane = threadIdx.x & 63;
  const long row = pair / heads;
  const int h = (int)(pair % heads);
  if (row >= start[num_segs]) return;
  if (skip_from > 0) {
    int lo_s = 0, hi_s = num_segs;
    while (hi_s - lo_s > 1) {
      const int mid = (lo_s + hi_s) >> 1;
      if (start[mid] <= row) lo_s = mid; else hi_s = mid;
    }
    if (start[lo_s + 1] - start[lo_s] >= skip_from) return;
  }
  // lane = slice (splits <= 64)
  const long b0 = row * splits * heads + h;
  float ms = -INFINITY, ls = 0.f;
  if (lane < splits) {
    ms = ws_ml[(b0 + (long)lane * heads) * 2];
    ls = ws_ml[(b0 + (long)lane * heads) * 2 + 1];
  }
  const float M = ft::wave_max(ms);
  const float w = ms == -INFINITY ? 0.f : expf(ms - M);
  const float L = ft::wave_sum(w * ls);
  const float inv = L > 0.f ? 1.0f / L : 0.f;
  for (int c = lane; c - lane < dv; c += 64) {
    float v = 0.f;
#pragma unroll 4
    for (int sp = 0; sp < splits; ++sp) {
      const float ws = __shfl(w, sp);
      if (c < dv) v += ws * ws_acc[(b0 + (long)sp * heads) * dv + c];
    }
    if (c < dv) {
      v *= inv;
      if (gate != nullptr) v *= sigmoidf_(ld(gate, row * gate_stride + (long)h * dv + c));
      st(out, (row * heads + h) * dv + c, v);
    }
  }
}

// ---------------------------------------------------------------------------------
// dot products -> unnormalised weights, in place, for the banded products: S [heads][rows]
// [keys], one workgroup of four waves per row (all heads).  The first `ext` columns are the
// positions 0 .. ext-1, column c >= ext is position key0 + c - ext.
// The mix over the heads runs on the matrix units in fp32 (v_mfma_f32_16x16x4_f32): for 16
// columns, lane (quarter q, column n) holds the capped scores of heads 16 b + 4 q + i, the
// k-step (b, i) of the product sums over the quarters, and the result lands in the same
// places (heads 16 b + 4 q + r).  inv [heads][rows] = 1 / row sum.  NB = ceil(heads / 16).
// ---------------------------------------------------------------------------------
typedef float f32x4_t __attribute__((ext_vector_type(4)));

template <int NB>
__global__ void __launch_bounds__(256)
talk_weights_kernel(float* __restrict__ S, float* __restrict__ inv, int heads, int rows, int keys, int first_pos,
                    int key0, int ext, int window, int keep_first, float softcap, const float* __restrict__ talk) {
  __shared__ float red[4][NB * 16];
  const int t = blockIdx.x, i = first_pos + t;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int n = lane & 15, qt = lane >> 4;
  const long hs = (long)rows * keys;               // from one head's scores to the next one's
  float* sp = S + (long)t * keys;
  // the mix as the left operand: row 16 ob + n, k-step (ib, u) is head 16 ib + 4 qt + u
  float tm[NB][NB][4];
#pragma unroll
  for (int ob = 0; ob < NB; ++ob)
#pragma unroll
    for (int ib = 0; ib < NB; ++ib)
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int h = 16 * ob + n, g = 16 * ib + 4 * qt + u;
        tm[ob][ib][u] = h < heads && g < heads ? talk[(long)h * heads + g] : 0.f;
      }
  auto visible = [&](int c) {
    const int p = c < ext ? c : key0 + c - ext;
    return c < keys && p <= i && (window <= 0 || i - p < window || p < keep_first);
  };
  float mx_[NB * 4];
#pragma unroll
  for (int u = 0; u < NB * 4; ++u) mx_[u] = -INFINITY;
  const int groups = (keys + 15) / 16;
  for (int gr = wave; gr < groups; gr += 4) {
    const int c = gr * 16 + n;
    const bool vis = visible(c);
    if (__ballot(vis) == 0) continue;              // (wave-uniform)
    float sc[NB][4];
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int h = 16 * b + 4 * qt + u;
        sc[b][u] = vis && h < heads ? sp[h * hs + c] : 0.f;
      }
    if (softcap > 0.f) {
#pragma unroll
      for (int b = 0; b < NB; ++b)
#pragma unroll
        for (int u = 0; u < 4; ++u) sc[b][u] = softcap * tanhf(sc[b][u] / softcap);
    }
#pragma unroll
    for (int ob = 0; ob < NB; ++ob) {
      f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ib = 0; ib < NB; ++ib)
#pragma unroll
        for (int u = 0; u < 4; ++u)
          acc = __builtin_amdgcn_mfma_f32_16x16x4f32(tm[ob][ib][u], sc[ib][u], acc, 0, 0, 0);
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int h = 16 * ob + 4 * qt + u;
        if (vis && h < heads) {
          sp[h * hs + c] = acc[u];                 // each lane re-reads only its own entries
          mx_[4 * ob + u] = fmaxf(mx_[4 * ob + u], acc[u]);
        }
      }
    }
  }
  // a head's maximum: over the 16 columns' lanes, then over the waves
#pragma unroll
  for (int u = 0; u < NB * 4; ++u) {
    mx_[u] = ft::group_max<16>(mx_[u]);
    if (n == 0) red[wave][16 * (u / 4) + 4 * qt + u % 4] = mx_[u];
  }
  __syncthreads();
#pragma unroll
  for (int u = 0; u < NB * 4; ++u) {
    const int h = 16 * (u / 4) + 4 * qt + u % 4;
    mx_[u] = fmaxf(fmaxf(red[0][h], red[1][h]), fmaxf(red[2][h], red[3][h]));
  }
  float sum[NB * 4];
#pragma unroll
  for (int u = 0; u < NB * 4; ++u) sum[u] = 0.f;
  for (int gr = wave; gr < groups; gr += 4) {
    const int c = gr * 16 + n;
    if (c >= keys) continue;
    const bool vis = visible(c);
#pragma unroll
    for (int u = 0; u < NB * 4; ++u) {
      const int h = 16 * (u / 4) + 4 * qt + u % 4;
      if (h < heads) {
        const float p = vis ? expf(sp[h * hs + c] - mx_[u]) : 0.f;
        sp[h * hs + c] = p;
        sum[u] += p;
      }
    }
  }
  __syncthreads();                                 // red was read above
#pragma unroll
  for (int u = 0; u < NB * 4; ++u) {
    sum[u] = ft::group_sum<16>(sum[u]);
    if (n == 0) red[wave][16 * (u / 4) + 4 * qt + u % 4] = sum[u];
  }
  __syncthreads();
  for (int h = threadIdx.x; h < heads; h += 256) {
    const float v = red[0][h] + red[1][h] + red[2][h] + red[3][h];
    inv[(long)h * rows + t] = v > 0.f ? 1.0f / v : 0.f;
  }
}

// out[t][h dv + c] = o[h][t][c] (* inv[h][t]) (* sigmoid(gate)), gate one number per row and
// head (per_head) or per element; per-head results become rows of the output projection
template <typename TG, typename TO>
__global__ void heads_to_rows_kernel(TO* __restrict__ out, const float* __restrict__ o, const float* __restrict__ inv,
                                     const TG* __restrict__ gate, long gate_stride, int per_head, long rows,
                                     int heads, int dv) {
  const long n = (long)heads * dv, total = rows * n;
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (long)gridDim.x * blockDim.x) {
    const long t = i / n;
    const int e = (int)(i % n), h = e / dv;
    float v = o[((long)h * rows + t) * dv + e % dv];
    if (inv != nullptr) v *= inv[(long)h * rows + t];
    if (gate != nullptr) v *= sigmoidf_(ld(gate, t * gate_stride + (per_head ? h : e)));
    st(out, i, v);
  }
}

}  // namespace mx

using namespace mx;

extern "C" int mx_rot_norm_prep(float* q_out, const void* qk, int bf16, long stride, int q_heads, int k_heads,
                                int head_dim, const float* table, int table_rows, int rot_dims, int interleaved,
                                float eps, const float* q_scale, const int* positions, const int* slots,
                                void* k_cache, void* v_cache, long num_slots, long rows, hipStream_t s) {
  if (rows <= 0) return 0;
  if (head_dim < 1 || head_dim > 64 * kPrepCols || rot_dims < 0 || rot_dims > head_dim || rot_dims % 2) return -1;
  if (rows > 0x7fffffffL || (q_heads + k_heads + 3) / 4 > 65535) return -2;
  const dim3 grid((unsigned)rows, (unsigned)((q_heads + k_heads + 3) / 4));
  MX_DISPATCH_T(bf16, hipLaunchKernelGGL((rot_norm_prep_kernel<T, T>), grid, dim3(256), 0, s, q_out, (const T*)qk,
                                         stride, q_heads, k_heads, head_dim, table, table_rows, rot_dims,
                                         interleaved, eps, q_scale, positions, slots, (T*)k_cache, (T*)v_cache,
                                         num_slots));
  return (int)hipGetLastError();
}

extern "C" int mx_talk_max_heads() { return 64; }

template <typename TC, int HPW, int HU>
static void launch_talk(bool vecv, dim3 grid, size_t shm, hipStream_t s, float* ws_acc, float* ws_ml, const float* q,
                        const void* k_cache, const void* v_cache, const int* start, const int* pos0,
                        const int* kv_len, const int* bt, int bt_stride, int num_segs, int heads, int kv_heads,
                        int dk, int dv, int window, int keep_first, float softcap, const float* talk,
                        int block_size, int num_blocks, int skip_from, int splits, int vec, int lpk) {
#define MX_TALK(V)                                                                                              \
  hipLaunchKernelGGL((talk_attn_kernel<TC, HPW, HU, V>), grid, dim3(64 * kTalkWaves), shm, s, ws_acc, ws_ml, q, \
                     (const TC*)k_cache, (const TC*)v_cache, start, pos0, kv_len, bt, bt_stride, num_segs,      \
                     heads, kv_heads, dk, dv, window, keep_first, softcap, talk, block_size, num_blocks,        \
                     skip_from, splits, vec, lpk)
  if (vecv) MX_TALK(true);
  else MX_TALK(false);
#undef MX_TALK
}

extern "C" int mx_talk_attention(void* out, int out_bf16, float* ws_acc, float* ws_ml, const float* q,
                                 const void* gate, long gate_stride, const void* k_cache, const void* v_cache,
                                 int cache_bf16, const int* start, const int* pos0, const int* kv_len, const int* bt,
                                 int bt_stride, int num_segs, long total_rows, int heads, int kv_heads, int dk,
                                 int dv, int window, int keep_first, float softcap, const float* talk,
                                 int block_size, int num_blocks, int skip_from, int splits, hipStream_t s) {
  if (num_segs <= 0 || total_rows <= 0) return 0;
  if (heads < 1 || heads > mx_talk_max_heads() || kv_heads < 1 || heads % kv_heads || dk < 1 || dv < 1 ||
      dv > 64 * kScalarCols || keep_first < 0 || splits < 1 || splits > 64)
    return -1;
  if (total_rows * splits > 0x7fffffffL || total_rows * heads > 0x7fffffffL) return -2;
  const size_t shm = (size_t)(heads * dk + 2 * heads * kTalkTile) * sizeof(float);
  if (shm > 64 * 1024) return -3;
  const long es = cache_bf16 ? 2 : 4;
  const int vec = (dk * es) % 16 == 0 && ((uintptr_t)k_cache) % 16 == 0;
  const long pieces = dv * es / 16;
  const bool vecv = (dv * es) % 16 == 0 && ((uintptr_t)v_cache) % 16 == 0 && pieces <= 64;
  int lpk = 1;
  while (lpk < pieces) lpk <<= 1;
  if (!vecv) lpk = 1;
  const int rep = heads / kv_heads, hpw = (heads + kTalkWaves - 1) / kTalkWaves;
  const dim3 grid((unsigned)(total_rows * splits));
#define MX_TL(W, U)                                                                                              \
  MX_DISPATCH_T(cache_bf16, (launch_talk<T, W, U>(vecv, grid, shm, s, ws_acc, ws_ml, q, k_cache, v_cache, start, \
                                                  pos0, kv_len, bt, bt_stride, num_segs, heads, kv_heads, dk, dv, \
                                                  window, keep_first, softcap, talk, block_size, num_blocks,      \
                                                  skip_from, splits, vec, lpk)))
#define MX_TU(W)           \
  do {                     \
    if (rep <= 1) MX_TL(W, 1);      \
    else if (rep <= 2) MX_TL(W, 2); \
    else MX_TL(W, 4);               \
  } while (0)
  if (hpw <= 1) MX_TU(1);
  else if (hpw <= 2) MX_TU(2);
  else if (hpw <= 4) MX_TU(4);
  else if (hpw <= 8) MX_TU(8);
  else MX_TU(16);
#undef MX_TU
#undef MX_TL
  const unsigned g2 = (unsigned)((total_rows * heads + 3) / 4);
  MX_DISPATCH_T(out_bf16, hipLaunchKernelGGL((talk_combine_kernel<T, T>), dim3(g2), dim3(256), 0, s, (T*)out, ws_acc,
                                             ws_ml, (const T*)gate, gate_stride, start, num_segs, total_rows, heads,
                                             dv, skip_from, splits));
  return (int)hipGetLastError();
}

extern "C" int mx_talk_weights(float* S, float* inv, int heads, int rows, int keys, int first_pos, int key0, int ext,
                               int window, int keep_first, float softcap, const float* talk, hipStream_t s) {
  if (heads <= 0 || rows <= 0 || keys <= 0) return 0;
  if (heads > mx_talk_max_heads() || keep_first < 0 || ext < 0 || ext > keys || ext > key0 || first_pos < 0) return -1;
  const dim3 grid((unsigned)rows), block(256);
#define MX_TW(NB)                                                                                              \
  hipLaunchKernelGGL((talk_weights_kernel<NB>), grid, block, 0, s, S, inv, heads, rows, keys, first_pos, key0, ext, \
                     window, keep_first, softcap, talk)
  if (heads <= 16) MX_TW(1);
  else if (heads <= 32) MX_TW(2);
  else MX_TW(4);
#undef MX_TW
  return (int)hipGetLastError();
}

extern "C" int mx_heads_to_rows(void* out, int out_bf16, const float* o, const float* inv, const void* gate,
                                long gate_stride, int per_head, long rows, int heads, int dv, hipStream_t s) {
  const long total = rows * heads * dv;
  if (total <= 0) return 0;
  long g = (total + 255) / 256;
  if (g > 65535) g = 65535;
  MX_DISPATCH_T(out_bf16, hipLaunchKernelGGL((heads_to_rows_kernel<T, T>), dim3((unsigned)g), dim3(256), 0, s,
                                             (T*)out, o, inv, (const T*)gate, gate_stride, per_head, rows, heads, dv));
  return (int)hipGetLastError();
}
