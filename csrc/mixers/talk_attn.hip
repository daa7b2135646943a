// Grouped-query attention that mixes its scores across the heads before the softmax, over a
// paged key cache and a paged value cache.
//
// Query head h reads key and value head h / rep, rep = heads / kv_heads.  Position i sees
// key j iff j <= i and (i - j < window, or window == 0, or j < keep_first).  With dot
// products s_g = q_g . k (queries come scaled): s_g <- softcap tanh(s_g / softcap) when
// softcap > 0, z_h = sum_g talk[h][g] s_g, weights = softmax of z_h over the visible keys;
// optionally with a sink, one more term exp(sink) (sinks[h], or the same for all heads) in the
// denominator.  Without `talk` the scores are not mixed (z = s): plain grouped-query attention
// on the same tiles.
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
// decode rows and short segments: one workgroup of W = 4 or 8 waves per (row, slice of its
// keys), 64 keys per tile.
//   scores: TILED (bf16 keys, rows of whole 16-byte pieces): wave w takes keys 16 (w mod 4) ..
//           + 15 and, of eight waves, every second group of four key heads (w / 4); for each key head, all query heads times the 16 keys on the matrix units
//           (v_mfma_f32_16x16x32_bf16) with the queries split into three bf16 parts, hi + mid +
//           lo, so that the products are those of the fp32 queries; a lane (quarter q, column n)
//           ends with the scores of heads 16 b + 4 q + u for key n.  Otherwise lane = key, a
//           wave takes groups of query heads that share a key head, and the scores change hands
//           through LDS.
//   mix:    cap, then the head mix on the matrix units in fp32 (v_mfma_f32_16x16x4_f32): the
//           k-step (b, u) of the product sums over the quarters, and a result lands where the
//           score of its head was; of eight waves, two leave partial results (heads they have no
//           scores of count as zeros) that are added when they are read
//   softmax: a wave owns HPW consecutive heads, 16 lanes per head with four keys each
//   sums:   a lane owns one 16-byte piece of the value row of every (64 / LPK)-th key, as in
//           window_attn_kernel, for all of the wave's heads at once (VEC), or lane = column.
//           AHEAD = LPK = 8 or 16 (all heads of a wave share a value head): the
//           tile's value pieces are all loaded as soon as the key pieces have been used, and
//           travel while the scores are capped, mixed and turned into weights
// Each slice leaves (max, sum, weighted sums) per head for talk_combine_kernel.
// ---------------------------------------------------------------------------------
constexpr int kTalkTile = 64;

typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));

template <typename TC> struct Row16;
template <> struct Row16<float> {
  static constexpr int N = 4;
  static __device__ __forceinline__ void widen(const uint4& u, float* v) {
    v[0] = __uint_as_float(u.x);
    v[1] = __uint_as_float(u.y);
    v[2] = __uint_as_float(u.z);
    v[3] = __uint_as_float(u.w);
  }
};
template <> struct Row16<bf16_t> {
  static constexpr int N = 8;
  static __device__ __forceinline__ void widen(const uint4& u, float* v) {
    const uint32_t w[4] = {u.x, u.y, u.z, u.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      v[2 * i] = __uint_as_float(w[i] << 16);
      v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
  }
};

template <typename TC>
__device__ __forceinline__ uint4 piece16(const TC* p) {
  return *reinterpret_cast<const uint4*>(p);
}

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

// the head mix as the left operand of the 16x16x4 fp32 product: row 16 ob + n of the mix,
// k-step (ib, u) is head 16 ib + 4 qt + u of this lane's quarter qt.  Entries past the last
// head repeat other entries: they meet scores that are zero, or leave results no one reads.
template <int NB>
__device__ __forceinline__ void load_mix(float (&tm)[NB][NB][4], const float* __restrict__ talk, int heads, int n,
                                         int qt) {
#pragma unroll
  for (int ob = 0; ob < NB; ++ob)
#pragma unroll
    for (int ib = 0; ib < NB; ++ib) {
      const int g = 16 * ib + 4 * qt;
      const float* row = talk + (long)min(16 * ob + n, heads - 1) * heads;
      if (heads % 4 == 0) {                         // (uniform; rows of whole 16-byte pieces)
        const float4 t = *reinterpret_cast<const float4*>(row + min(g, heads - 4));
        tm[ob][ib][0] = t.x; tm[ob][ib][1] = t.y; tm[ob][ib][2] = t.z; tm[ob][ib][3] = t.w;
      } else {
#pragma unroll
        for (int u = 0; u < 4; ++u) tm[ob][ib][u] = row[min(g + u, heads - 1)];
      }
    }
}

template <int NB>
__device__ __forceinline__ f32x4_t mix_block(const float (&tm)[NB][NB][4], const float (&sc)[NB][4], int ob) {
  f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int ib = 0; ib < NB; ++ib)
#pragma unroll
    for (int u = 0; u < 4; ++u) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(tm[ob][ib][u], sc[ib][u], acc, 0, 0, 0);
  return acc;
}

constexpr int kScalarCols = 8;                // value columns per lane (scalar form): dv <= 512
constexpr int kShareHeads = 4;                // query heads that read a key row together (not TILED)

// elements of a query row in LDS, TILED: whole steps of 32, plus 8 so that the 16 rows a wave
// reads at once fall on different banks
__host__ __device__ constexpr int tiled_row(int dk) { return (dk + 31) / 32 * 32 + 8; }

template <typename TC, int W, int HPW, bool TILED, bool VEC, int AHEAD>
__global__ void __launch_bounds__(64 * W)
talk_attn_kernel(float* __restrict__ ws_acc, float* __restrict__ ws_ml, const float* __restrict__ q,
                 const TC* __restrict__ k_cache, const TC* __restrict__ v_cache, const int* __restrict__ start,
                 const int* __restrict__ pos0, const int* __restrict__ kv_len, const int* __restrict__ bt,
                 int bt_stride, int num_segs, int heads, int kv_heads, int dk, int dv, int window, int keep_first,
                 float softcap, const float* __restrict__ talk, float q_mult, int block_size, int num_blocks,
                 int skip_from, int splits, int vec, int lpk) {
  constexpr int CAP = W * HPW;                       // heads there is room for
  constexpr int NB = (CAP + 15) / 16;                // 16-head blocks
  constexpr int RND = (HPW + 3) / 4;                 // softmax rounds of a wave (four heads each)
  extern __shared__ float smem[];
  const long row = blockIdx.x / splits;
  const int sp = blockIdx.x % splits;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int n = lane & 15, qt = lane >> 4;
  if (row >= start[num_segs]) return;
  const int s = segment_of(start, num_segs, (int)row);
  const int r0 = start[s], rows_s = start[s + 1] - r0;
  if (skip_from > 0 && rows_s >= skip_from) return;
  const long nk = (long)kv_heads * dk, nv = (long)kv_heads * dv;
  const TalkBand b = talk_band(pos0[s] + (int)(row - r0), kv_len[s], window, keep_first);
  const int tiles = (b.nkeys + kTalkTile - 1) / kTalkTile;
  const int per = (tiles + splits - 1) / splits * kTalkTile;
  const int begin = min(sp * per, b.nkeys), end = min(begin + per, b.nkeys);
  const int* table = bt + (long)s * bt_stride;
  const int rep = heads / kv_heads;
  // page of key index c (-1: none): loaded a tile ahead, the first one before anything else
  auto page_of = [&](int c) {
    const int j = c < b.ext ? c : b.first + c - b.ext;
    return c < end ? table[j / block_size] : -1;
  };
  int blk = page_of(begin + lane);
  float* z_s = smem;                                 // [W / 4][CAP][64] mixed scores; then each wave's weights [64][HPW]
  float* q_s = smem + W / 4 * CAP * kTalkTile;           // fp32 [heads][dk], or bf16 [3][16 NB][tiled_row(dk)]
  const float* qp = q + row * (long)heads * dk;
  const int qrow = tiled_row(dk);
  if constexpr (TILED) {
    // four entries per load, several loads in flight
    bf16_t* qb = reinterpret_cast<bf16_t*>(q_s);
    const int part = 16 * NB * qrow, q4 = dk / 4, total = heads * q4;
    constexpr int QL = 4;
    for (int e0 = tid; e0 < total; e0 += 64 * W * QL) {
      float4 v4[QL];
#pragma unroll
      for (int x = 0; x < QL; ++x)
        if (e0 + 64 * W * x < total) v4[x] = *reinterpret_cast<const float4*>(qp + 4 * (e0 + 64 * W * x));
#pragma unroll
      for (int x = 0; x < QL; ++x) {
        const int e = e0 + 64 * W * x;
        if (e < total) {
          const float v[4] = {v4[x].x * q_mult, v4[x].y * q_mult, v4[x].z * q_mult, v4[x].w * q_mult};
          float r1[4], r2[4];
          uint32_t p0[2], p1[2], p2[2];
#pragma unroll
          for (int k = 0; k < 4; ++k) r1[k] = v[k] - ft::bf16_to_f32(ft::f32_to_bf16(v[k]));
#pragma unroll
          for (int k = 0; k < 4; ++k) r2[k] = r1[k] - ft::bf16_to_f32(ft::f32_to_bf16(r1[k]));
#pragma unroll
          for (int k = 0; k < 2; ++k) {
            p0[k] = ft::pack2(v[2 * k], v[2 * k + 1]);
            p1[k] = ft::pack2(r1[2 * k], r1[2 * k + 1]);
            p2[k] = ft::pack2(r2[2 * k], r2[2 * k + 1]);
          }
          const int h = e / q4;
          bf16_t* dst = qb + h * qrow + 4 * (e - h * q4);
          *reinterpret_cast<uint2*>(dst) = make_uint2(p0[0], p0[1]);
          *reinterpret_cast<uint2*>(dst + part) = make_uint2(p1[0], p1[1]);
          *reinterpret_cast<uint2*>(dst + 2 * part) = make_uint2(p2[0], p2[1]);
        }
      }
    }
    // zeros past the last head and past a row's last entry
    if (heads < 16 * NB)
      for (int e = heads * qrow + tid; e < part; e += 64 * W) qb[e] = qb[part + e] = qb[2 * part + e] = 0;
    if (dk % 32)
      for (int e = tid; e < heads * 32; e += 64 * W) {
        const int d = dk + e % 32;
        if (d < qrow) {
          bf16_t* dst = qb + (e / 32) * qrow + d;
          dst[0] = dst[part] = dst[2 * part] = 0;
        }
      }
  } else {
    for (int d = tid; d < heads * dk; d += 64 * W) q_s[d] = qp[d] * q_mult;
  }
  float tm[NB][NB][4];
  if (talk != nullptr) load_mix<NB>(tm, talk, heads, n, qt);
  const int col = 16 * (wave & 3) + n, half = wave >> 2;   // the key and the share of the heads it scores
  const int h0 = wave * HPW;                         // this wave's heads h0 .. h0 + HPW - 1 (< heads)
  // the key head of each score this lane holds (-1: no such head)
  int kh[NB][4];
#pragma unroll
  for (int bb = 0; bb < NB; ++bb)
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int h = 16 * bb + 4 * qt + u;
      kh[bb][u] = h < heads ? h / rep : -1;
    }

  constexpr int NO = VEC ? Row16<TC>::N : kScalarCols;
  float o[HPW][NO], m[RND], l[RND];
#pragma unroll
  for (int x = 0; x < HPW; ++x)
#pragma unroll
    for (int u = 0; u < NO; ++u) o[x][u] = 0.f;
#pragma unroll
  for (int r = 0; r < RND; ++r) {
    m[r] = -INFINITY;
    l[r] = 0.f;
  }
  const int pieces = dv / Row16<TC>::N;
  if constexpr (AHEAD > 0) lpk = AHEAD;
  const int sg = lane & (lpk - 1), sub = lane / lpk, kpp = 64 / lpk;
  const bool has_piece = sg < pieces;
  for (int c0 = begin; c0 < end; c0 += kTalkTile) {
    const int cc = c0 + lane;
    const int j = cc < b.ext ? cc : b.first + cc - b.ext;
    const int slot = blk >= 0 && blk < num_blocks ? blk * block_size + j % block_size : -1;
    blk = page_of(cc + kTalkTile);
    const int slot16 = __shfl(slot, col);      // the key whose scores this lane holds
    __syncthreads();                                 // q_s is there / the last tile's z_s is no longer read
    // AHEAD: this lane's value pieces of the tile (pass ps: key ps * kpp + sub)
    uint4 vr[AHEAD > 0 ? AHEAD : 1];
    auto load_values = [&]() {
      const TC* vp = v_cache + (long)(min(h0, heads - 1) / rep) * dv + min(sg, pieces - 1) * Row16<TC>::N;
#pragma unroll
      for (int ps = 0; ps < AHEAD; ++ps) vr[ps] = piece16(vp + (long)max(__shfl(slot, ps * kpp + sub), 0) * nv);
    };
    float sc[NB][4];
#pragma unroll
    for (int bb = 0; bb < NB; ++bb)
#pragma unroll
      for (int u = 0; u < 4; ++u) sc[bb][u] = 0.f;
    if constexpr (TILED) {
      const bf16_t* qb = reinterpret_cast<const bf16_t*>(q_s) + n * qrow + 8 * qt;
      const int part = 16 * NB * qrow;
      const bf16_t* kp = reinterpret_cast<const bf16_t*>(k_cache) + (long)max(slot16, 0) * nk;
      for (int g0 = 4 * half; g0 < kv_heads; g0 += W) {
        f32x4_t acc[NB][4];
#pragma unroll
        for (int bb = 0; bb < NB; ++bb)
#pragma unroll
          for (int gi = 0; gi < 4; ++gi) acc[bb][gi] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        for (int d0 = 0; d0 < dk; d0 += 128) {
          uint4 kr[4][4];
#pragma unroll
          for (int gi = 0; gi < 4; ++gi)
#pragma unroll
            for (int st = 0; st < 4; ++st) {
              // entries past the row's end meet zeros of the queries, key heads past the last no score
              const int d = min(d0 + 32 * st + 8 * qt, dk - 8);
              kr[gi][st] = piece16(kp + (long)min(g0 + gi, kv_heads - 1) * dk + d);
            }
#pragma unroll
          for (int bb = 0; bb < NB; ++bb) {
            // key heads g0 .. g0 + 3 serve query heads g0 rep .. (g0 + 4) rep - 1
            if (g0 * rep >= 16 * bb + 16 || (g0 + 4) * rep <= 16 * bb) continue;
#pragma unroll
            for (int st = 0; st < 4; ++st) {
              if (d0 + 32 * st >= dk) break;
              const bf16_t* qa = qb + 16 * bb * qrow + d0 + 32 * st;
              const bf16x8_t q0 = __builtin_bit_cast(bf16x8_t, piece16(qa));
              const bf16x8_t q1 = __builtin_bit_cast(bf16x8_t, piece16(qa + part));
              const bf16x8_t q2 = __builtin_bit_cast(bf16x8_t, piece16(qa + 2 * part));
#pragma unroll
              for (int gi = 0; gi < 4; ++gi) {
                const bf16x8_t kf = __builtin_bit_cast(bf16x8_t, kr[gi][st]);
                f32x4_t a = acc[bb][gi];
                a = __builtin_amdgcn_mfma_f32_16x16x32_bf16(q2, kf, a, 0, 0, 0);
                a = __builtin_amdgcn_mfma_f32_16x16x32_bf16(q1, kf, a, 0, 0, 0);
                acc[bb][gi] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(q0, kf, a, 0, 0, 0);
              }
            }
          }
        }
#pragma unroll
        for (int bb = 0; bb < NB; ++bb)
#pragma unroll
          for (int gi = 0; gi < 4; ++gi)
#pragma unroll
            for (int u = 0; u < 4; ++u)
              if (kh[bb][u] == g0 + gi) sc[bb][u] = acc[bb][gi][u];
      }
    } else {
      const TC* krow = k_cache + (long)max(slot, 0) * nk;
      const int upg = (rep + kShareHeads - 1) / kShareHeads, units = kv_heads * upg;
      for (int un = wave; un < units; un += W) {
        const int g = un / upg, x0 = (un % upg) * kShareHeads, hb = g * rep + x0;
        const int nh = min(kShareHeads, rep - x0);
        const TC* kp = krow + (long)g * dk;
        float acc[kShareHeads];
        const float* qh[kShareHeads];
#pragma unroll
        for (int x = 0; x < kShareHeads; ++x) {
          acc[x] = 0.f;
          qh[x] = q_s + (long)(hb + min(x, nh - 1)) * dk;
        }
        if (vec) {
          constexpr int N = Row16<TC>::N;
#pragma unroll 8
          for (int d = 0; d < dk; d += N) {
            float kv[N];
            Row16<TC>::widen(piece16(kp + d), kv);
#pragma unroll
            for (int x = 0; x < kShareHeads; ++x)
#pragma unroll
              for (int f = 0; f < N; f += 4) {
                const float4 q4 = *reinterpret_cast<const float4*>(qh[x] + d + f);
                acc[x] += q4.x * kv[f] + q4.y * kv[f + 1] + q4.z * kv[f + 2] + q4.w * kv[f + 3];
              }
          }
        } else {
          for (int d = 0; d < dk; ++d) {
            const float kv = ld(kp, d);
#pragma unroll
            for (int x = 0; x < kShareHeads; ++x) acc[x] += qh[x][d] * kv;
          }
        }
#pragma unroll
        for (int x = 0; x < kShareHeads; ++x)
          if (x < nh) z_s[(hb + x) * kTalkTile + lane] = acc[x];
      }
      __syncthreads();
      // from here on a wave touches only its own 16 columns until the next barrier
#pragma unroll
      for (int bb = 0; bb < NB; ++bb)
#pragma unroll
        for (int u = 0; u < 4; ++u)
          if (kh[bb][u] >= 0 && half == 0) sc[bb][u] = z_s[(16 * bb + 4 * qt + u) * kTalkTile + col];
    }
    if constexpr (AHEAD > 0) load_values();
    if (softcap > 0.f) {
#pragma unroll
      for (int bb = 0; bb < NB; ++bb)
#pragma unroll
        for (int u = 0; u < 4; ++u) sc[bb][u] = softcap * tanh_(sc[bb][u] / softcap);
    }
#pragma unroll
    for (int bb = 0; bb < NB; ++bb) {
      f32x4_t z = {sc[bb][0], sc[bb][1], sc[bb][2], sc[bb][3]};
      if (talk != nullptr) z = mix_block<NB>(tm, sc, bb);
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (kh[bb][u] >= 0)
          z_s[(half * CAP + 16 * bb + 4 * qt + u) * kTalkTile + col] = slot16 >= 0 ? z[u] : -INFINITY;
    }
    __syncthreads();
    if (h0 < heads) {
      // 16 lanes per head, four keys per lane; all of the wave's scores are read before its
      // region of z_s is written over with the weights, keys outermost
      float z[RND][4], resc[RND];
#pragma unroll
      for (int r = 0; r < RND; ++r) {
        const int x = 4 * r + qt;
        const bool on = x < HPW && h0 + x < heads;
        float4 z4 = *reinterpret_cast<const float4*>(z_s + (h0 + (on ? x : 0)) * kTalkTile + 4 * n);
        if constexpr (W == 8) {
          const float4 y4 = *reinterpret_cast<const float4*>(z_s + (CAP + h0 + (on ? x : 0)) * kTalkTile + 4 * n);
          z4.x += y4.x; z4.y += y4.y; z4.z += y4.z; z4.w += y4.w;
        }
        z[r][0] = z4.x; z[r][1] = z4.y; z[r][2] = z4.z; z[r][3] = z4.w;
        const float mn = fmaxf(m[r], max16(fmaxf(fmaxf(z4.x, z4.y), fmaxf(z4.z, z4.w))));
        resc[r] = m[r] == -INFINITY ? 0.f : expf(m[r] - mn);
        float sum = 0.f;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          z[r][e] = on && z[r][e] != -INFINITY ? expf(z[r][e] - mn) : 0.f;
          sum += z[r][e];
        }
        l[r] = l[r] * resc[r] + sum16(sum);
        m[r] = mn;
      }
      wave_lds_fence();
      float* p_s = z_s + h0 * kTalkTile;             // [64][HPW]
#pragma unroll
      for (int r = 0; r < RND; ++r) {
        const int x = 4 * r + qt;
        if (x < HPW) {
#pragma unroll
          for (int e = 0; e < 4; ++e) p_s[(4 * n + e) * HPW + x] = z[r][e];
        }
      }
      wave_lds_fence();
      if (c0 > begin) {
#pragma unroll
        for (int x = 0; x < HPW; ++x) {
          const float f = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(resc[x / 4]), 16 * (x % 4)));
#pragma unroll
          for (int u = 0; u < NO; ++u) o[x][u] *= f;
        }
      }
      const int cnt = min(kTalkTile, end - c0);
      // weights past the tile's last key (and of heads past the last) are 0
      auto weights = [&](int key, float (&w)[HPW]) {
        if constexpr (HPW % 4 == 0) {
#pragma unroll
          for (int x = 0; x < HPW; x += 4) {
            const float4 w4 = *reinterpret_cast<const float4*>(p_s + key * HPW + x);
            w[x] = w4.x; w[x + 1] = w4.y; w[x + 2] = w4.z; w[x + 3] = w4.w;
          }
        } else {
#pragma unroll
          for (int x = 0; x < HPW; ++x) w[x] = p_s[key * HPW + x];
        }
      };
      if constexpr (AHEAD > 0) {
        // a lane past the row's last piece sums what is not stored
#pragma unroll
        for (int ps = 0; ps < AHEAD; ++ps) {
          float v[Row16<TC>::N], w[HPW];
          Row16<TC>::widen(vr[ps], v);
          weights(ps * kpp + sub, w);
#pragma unroll
          for (int x = 0; x < HPW; ++x)
#pragma unroll
            for (int u = 0; u < Row16<TC>::N; ++u) o[x][u] += w[x] * v[u];
        }
      } else if constexpr (VEC) {
        const int passes = (cnt + kpp - 1) / kpp;
#pragma unroll 4
        for (int ps = 0; ps < passes; ++ps) {
          const int jj = ps * kpp + sub;             // < 64
          const int sj = __shfl(slot, jj);
          const bool ok = sj >= 0 && has_piece;
          const TC* vrow = v_cache + (ok ? (long)sj * nv + sg * Row16<TC>::N : 0L);
          float v[Row16<TC>::N], w[HPW];
          weights(jj, w);
#pragma unroll
          for (int x = 0; x < HPW; ++x) {
            const int g = min(h0 + x, heads - 1) / rep;
            if (x == 0 || g != min(h0 + x - 1, heads - 1) / rep)
              Row16<TC>::widen(piece16(vrow + (ok ? (long)g * dv : 0L)), v);
#pragma unroll
            for (int u = 0; u < Row16<TC>::N; ++u) o[x][u] += (ok ? w[x] : 0.f) * v[u];
          }
        }
      } else {
        for (int jj = 0; jj < cnt; ++jj) {
          const int sj = __shfl(slot, jj);
          if (sj < 0) continue;
#pragma unroll
          for (int x = 0; x < HPW; ++x) {
            const TC* vp = v_cache + (long)sj * nv + (long)(min(h0 + x, heads - 1) / rep) * dv;
            const float w = p_s[jj * HPW + x];
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
      for (int off = lpk; off < 16; off <<= 1) {
#pragma unroll
        for (int u = 0; u < NO; ++u) o[x][u] += __shfl_xor(o[x][u], off);
      }
      if (lpk <= 16) {
#pragma unroll
        for (int u = 0; u < NO; ++u) o[x][u] = add_row_pair(o[x][u]);
      }
      if (lpk <= 32) {
#pragma unroll
        for (int u = 0; u < NO; ++u) o[x][u] = add_halves(o[x][u]);
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
    if (lane == 16 * (x % 4)) {
      ws_ml[(base + h) * 2] = m[x / 4];
      ws_ml[(base + h) * 2 + 1] = l[x / 4];
    }
  }
}

// one wave per (row, head, 256 columns): merges the slices, divides by the sum (with the sink's
// term, if there is one), applies the element-wise sigmoid gate (optional) and rounds
template <typename TG, typename TO, bool VEC>
__global__ void __launch_bounds__(256)
talk_combine_kernel(TO* __restrict__ out, const float* __restrict__ ws_acc, const float* __restrict__ ws_ml,
                    const TG* __restrict__ gate, long gate_stride, const int* __restrict__ start, int num_segs,
                    long total_rows, int heads, int dv, int skip_from, int splits, int has_sink, float sink_all,
                    const float* __restrict__ sinks) {
  const long pair = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (pair >= total_rows * heads) return;
  const int lane = threadIdx.x & 63;
  const long row = pair / heads;
  const int h = (int)(pair % heads);
  if (row >= start[num_segs]) return;
  if (skip_from > 0) {
    const int sg = segment_of(start, num_segs, (int)row);
    if (start[sg + 1] - start[sg] >= skip_from) return;
  }
  // lane = slice (splits <= 64)
  const long b0 = row * splits * heads + h;
  float ms = -INFINITY, ls = 0.f;
  if (lane < splits) {
    ms = ws_ml[(b0 + (long)lane * heads) * 2];
    ls = ws_ml[(b0 + (long)lane * heads) * 2 + 1];
  }
  float M = ft::wave_max(ms);
  const float sink = sinks != nullptr ? sinks[h] : sink_all;
  if (has_sink) M = fmaxf(M, sink);
  const float w = ms == -INFINITY ? 0.f : expf(ms - M);
  const float L = ft::wave_sum(w * ls) + (has_sink ? expf(sink - M) : 0.f);
  const float inv = L > 0.f ? 1.0f / L : 0.f;
  merge_slices<VEC>(ws_acc + b0 * dv, (long)heads * dv, w, splits, blockIdx.y * 256, dv, lane, [&](int c, float v) {
    v *= inv;
    if (gate != nullptr) v *= sigmoidf_(ld(gate, row * gate_stride + (long)h * dv + c));
    st(out, (row * heads + h) * dv + c, v);
  });
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
  float tm[NB][NB][4];
  load_mix<NB>(tm, talk, heads, n, qt);
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
        for (int u = 0; u < 4; ++u) sc[b][u] = softcap * tanh_(sc[b][u] / softcap);
    }
#pragma unroll
    for (int ob = 0; ob < NB; ++ob) {
      const f32x4_t acc = mix_block<NB>(tm, sc, ob);
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

template <typename TC, int W, int HPW>
static void launch_talk(bool tiled, bool vecv, int ahead, dim3 grid, size_t shm, hipStream_t s, float* ws_acc,
                        float* ws_ml, const float* q, const void* k_cache, const void* v_cache, const int* start,
                        const int* pos0, const int* kv_len, const int* bt, int bt_stride, int num_segs, int heads,
                        int kv_heads, int dk, int dv, int window, int keep_first, float softcap, const float* talk,
                        float q_mult, int block_size, int num_blocks, int skip_from, int splits, int vec, int lpk) {
#define MX_TALK(T, V, A)                                                                                        \
  hipLaunchKernelGGL((talk_attn_kernel<TC, W, HPW, T, V, A>), grid, dim3(64 * W), shm, s, ws_acc, ws_ml,  \
                     q, (const TC*)k_cache, (const TC*)v_cache, start, pos0, kv_len, bt, bt_stride, num_segs,   \
                     heads, kv_heads, dk, dv, window, keep_first, softcap, talk, q_mult, block_size, num_blocks, \
                     skip_from, splits, vec, lpk)
  if constexpr (sizeof(TC) == 2) {
    if (tiled && ahead == 16) MX_TALK(true, true, 16);
    else if (tiled && ahead == 8) MX_TALK(true, true, 8);
    else if (tiled) MX_TALK(true, true, 0);
    else MX_TALK(false, false, 0);
  } else {
    if (vecv) MX_TALK(false, true, 0);
    else MX_TALK(false, false, 0);
  }
#undef MX_TALK
}

extern "C" int mx_talk_attention(void* out, int out_bf16, float* ws_acc, float* ws_ml, const float* q,
                                 const void* gate, long gate_stride, const void* k_cache, const void* v_cache,
                                 int cache_bf16, const int* start, const int* pos0, const int* kv_len, const int* bt,
                                 int bt_stride, int num_segs, long total_rows, int heads, int kv_heads, int dk,
                                 int dv, int window, int keep_first, float softcap, const float* talk, float q_mult,
                                 int has_sink, float sink_all, const float* sinks, int block_size, int num_blocks,
                                 int skip_from, int splits, hipStream_t s) {
  if (num_segs <= 0 || total_rows <= 0) return 0;
  if (heads < 1 || heads > mx_talk_max_heads() || kv_heads < 1 || heads % kv_heads || dk < 1 || dv < 1 ||
      dv > 64 * kScalarCols || ((uintptr_t)talk) % 16 || ((uintptr_t)q) % 16 || keep_first < 0 || splits < 1 || splits > 64)
    return -1;
  if (total_rows * splits > 0x7fffffffL || total_rows * heads > 0x7fffffffL) return -2;
  const int rep = heads / kv_heads;
  const int waves = heads > 16 && heads <= 32 ? 8 : 4;
  int hpw = 1;                                         // heads per wave
  while (hpw * waves < heads) hpw <<= 1;
  const long es = cache_bf16 ? 2 : 4;
  const int vec = (dk * es) % 16 == 0 && ((uintptr_t)k_cache) % 16 == 0;
  const long pieces = dv * es / 16;
  const bool vecv = (dv * es) % 16 == 0 && ((uintptr_t)v_cache) % 16 == 0 && pieces <= 64;
  int lpk = 1;
  while (lpk < pieces) lpk <<= 1;
  const size_t z_bytes = (size_t)(waves / 4) * waves * hpw * kTalkTile * sizeof(float);
  const size_t tiled_bytes = z_bytes + (size_t)3 * ((waves * hpw + 15) / 16 * 16) * tiled_row(dk) * 2;
  const bool tiled = cache_bf16 && vec && vecv && tiled_bytes <= 64 * 1024;
  const size_t shm = tiled ? tiled_bytes : z_bytes + (size_t)heads * dk * sizeof(float);
  if (shm > 64 * 1024) return -3;
  if (!(vecv && (tiled || !cache_bf16))) lpk = 1;      // value columns lane by lane
  const int ahead = rep % hpw != 0 || pieces > 16 ? 0 : pieces > 8 ? 16 : 8;
  const dim3 grid((unsigned)(total_rows * splits));
#define MX_TL(W, H)                                                                                                  \
  MX_DISPATCH_T(cache_bf16, (launch_talk<T, W, H>(tiled, vecv, ahead, grid, shm, s, ws_acc, ws_ml, q, k_cache, v_cache, \
                                               start, pos0, kv_len, bt, bt_stride, num_segs, heads, kv_heads, dk,  \
                                               dv, window, keep_first, softcap, talk, q_mult, block_size, num_blocks, \
                                               skip_from, splits, vec, lpk)))
  if (waves == 8) MX_TL(8, 4);
  else if (hpw == 1) MX_TL(4, 1);
  else if (hpw == 2) MX_TL(4, 2);
  else if (hpw == 4) MX_TL(4, 4);
  else MX_TL(4, 16);
#undef MX_TL
  const dim3 g2((unsigned)((total_rows * heads + 3) / 4), (unsigned)((dv + 255) / 256));
#define MX_TC(V)                                                                                                \
  MX_DISPATCH_T(out_bf16, hipLaunchKernelGGL((talk_combine_kernel<T, T, V>), g2, dim3(256), 0, s, (T*)out,      \
                                             ws_acc, ws_ml, (const T*)gate, gate_stride, start, num_segs,       \
                                             total_rows, heads, dv, skip_from, splits, has_sink, sink_all, sinks))
  if (dv % 4 == 0 && ((uintptr_t)ws_acc) % 16 == 0) MX_TC(true);
  else MX_TC(false);
#undef MX_TC
  return (int)hipGetLastError();
}

extern "C" int mx_talk_weights(float* S, float* inv, int heads, int rows, int keys, int first_pos, int key0, int ext,
                               int window, int keep_first, float softcap, const float* talk, hipStream_t s) {
  if (heads <= 0 || rows <= 0 || keys <= 0) return 0;
  if (heads > mx_talk_max_heads() || ((uintptr_t)talk) % 16 || keep_first < 0 || ext < 0 || ext > keys || ext > key0 || first_pos < 0) return -1;
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
