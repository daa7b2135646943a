// Shared helpers of the sequence-mixer / MoE kernels (extension `_C_mixers`).
//
// Every kernel is instantiated for fp32 and bf16 activations (`T` = float or
// ft::bf16_raw); statistics, scores, recurrent state and gates are fp32 in both.
// Launchers take `int bf16` flags and void pointers, and the caller's stream.
#pragma once

#include <hip/hip_runtime.h>
#include <math.h>
#include <stdint.h>

#include "ft_common.h"

namespace mx {

using bf16_t = ft::bf16_raw;

__device__ __forceinline__ float ld(const float* p, long i) { return p[i]; }
__device__ __forceinline__ float ld(const bf16_t* p, long i) { return ft::bf16_to_f32(p[i]); }
__device__ __forceinline__ void st(float* p, long i, float v) { p[i] = v; }
__device__ __forceinline__ void st(bf16_t* p, long i, float v) { p[i] = ft::f32_to_bf16(v); }

__device__ __forceinline__ float sigmoidf_(float x) { return 1.0f / (1.0f + expf(-x)); }

// softplus with the usual linear branch for large arguments
__device__ __forceinline__ float softplusf_(float x) { return x > 20.0f ? x : log1pf(expf(x)); }

// entry d < dims of a head x after rotary positions, cs = [cos | sin] of the position: pairs
// (i, i + dims/2), or (2i, 2i + 1) if interleaved
template <typename T>
__device__ __forceinline__ float rope_at(const T* x, int d, int dims, const float* cs, int interleaved) {
  const int half = dims / 2;
  const int i = interleaved ? d >> 1 : (d < half ? d : d - half);
  const bool second = interleaved ? (d & 1) : d >= half;
  const int other = interleaved ? d ^ 1 : (second ? d - half : d + half);
  const float v = ld(x, d), w = ld(x, other), c = cs[i], s = cs[half + i];
  return second ? v * c + w * s : v * c - w * s;
}

// sum / maximum over the 16 lanes of a row (quad swaps, mirrored half row, mirrored row): every
// lane gets it
__device__ __forceinline__ float sum16(float v) {
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0xB1, 0xF, 0xF, true));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x4E, 0xF, 0xF, true));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x141, 0xF, 0xF, true));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x140, 0xF, 0xF, true));
  return v;
}
__device__ __forceinline__ float max16(float v) {
  v = fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0xB1, 0xF, 0xF, true)));
  v = fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x4E, 0xF, 0xF, true)));
  v = fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x141, 0xF, 0xF, true)));
  v = fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x140, 0xF, 0xF, true)));
  return v;
}

// v plus the v of the lane 16 / 32 away (row swaps instead of the LDS permute path)
__device__ __forceinline__ float add_row_pair(float v) {
  const auto r = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return __uint_as_float(r[0]) + __uint_as_float(r[1]);
}
__device__ __forceinline__ float add_halves(float v) {
  const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return __uint_as_float(r[0]) + __uint_as_float(r[1]);
}

// tanh without branches: the Taylor polynomial up to |x| = 1/4, (1 - e^-2|x|) / (1 + e^-2|x|) beyond
__device__ __forceinline__ float tanh_(float x) {
  const float a = fabsf(x), q = a * a;
  const float p = a + a * q * (-1.f / 3 + q * (2.f / 15 + q * (-17.f / 315 + q * (62.f / 2835 - q * (1382.f / 155925)))));
  const float t = __builtin_amdgcn_exp2f(-2.8853900817779268f * a);
  const float r = (1.f - t) / (1.f + t);
  return copysignf(a < 0.25f ? p : r, x);
}

// a wave's own LDS writes, to be read by its other lanes
__device__ __forceinline__ void wave_lds_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// the segment that owns a row: the last s with start[s] <= row.  Decode rows come first in a
// step, one row each: for them one look at two neighbouring entries is enough.
__device__ __forceinline__ int segment_of(const int* __restrict__ start, int num_segs, int row) {
  if (row < num_segs && start[row] == row && start[row + 1] == row + 1) return row;
  int lo = 0, hi = num_segs;
  while (hi - lo > 1) {
    const int mid = (lo + hi) >> 1;
    if (start[mid] <= row) lo = mid; else hi = mid;
  }
  return lo;
}

// A short causal convolution over time of one wave's channels c0 + lane + 64 u (u < NU, below
// c0 + len), walked row by row: taps (<= TAPS) weights and the last taps - 1 inputs in
// registers, fp32.  Missing taps in front count as zeros.
template <int TAPS, int NU>
struct ConvWalk {
  float w[NU][TAPS], win[NU][TAPS];            // win[u][TAPS - 1] is the current row's input

  __device__ __forceinline__ void weights(const float* __restrict__ conv_w, int taps, int c0, int len, int lane) {
    const int pad = TAPS - taps;
#pragma unroll
    for (int u = 0; u < NU; ++u) {
      const int i = lane + 64 * u;
      const float* p = conv_w + (long)(c0 + (i < len ? i : 0)) * taps;
      if (TAPS == 4 && pad == 0 && ((uintptr_t)conv_w) % 16 == 0) {
        const float4 v = *reinterpret_cast<const float4*>(p);
        w[u][0] = v.x; w[u][1] = v.y; w[u][TAPS == 4 ? 2 : 0] = v.z; w[u][TAPS == 4 ? 3 : 0] = v.w;
      } else {
#pragma unroll
        for (int j = 0; j < TAPS; ++j) w[u][j] = j >= pad ? p[j - pad] : 0.f;
      }
    }
  }
  // the inputs before row rel of the segment that starts at row r0: rows of x, further back the
  // history h [taps - 1][channels] (null: zeros)
  template <typename T>
  __device__ __forceinline__ void begin(const T* __restrict__ x, long stride, long r0, int rel, const float* h,
                                        int channels, int taps, int c0, int len, int lane) {
    const int pad = TAPS - taps;
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j) {
      const int src = rel - (TAPS - 1) + j;
#pragma unroll
      for (int u = 0; u < NU; ++u) {
        const int i = lane + 64 * u, c = c0 + (i < len ? i : 0);
        float v = 0.f;
        if (j >= pad) {
          if (src >= 0) v = ld(x, (r0 + src) * stride + c);
          else if (h != nullptr) v = h[(long)(taps - 1 + src) * channels + c];
        }
        win[u][j] = v;
      }
    }
  }
  __device__ __forceinline__ float step(int u, float v) {
    win[u][TAPS - 1] = v;
    float acc = 0.f;
#pragma unroll
    for (int j = 0; j < TAPS; ++j) acc += win[u][j] * w[u][j];
    return acc;
  }
  // to the next row
  __device__ __forceinline__ void shift(int u) {
#pragma unroll
    for (int j = 0; j + 1 < TAPS; ++j) win[u][j] = win[u][j + 1];
  }
  // after shift(): the last taps - 1 inputs, as a history
  __device__ __forceinline__ void store(float* h, int channels, int taps, int c0, int len, int lane) const {
    const int pad = TAPS - taps;
#pragma unroll
    for (int u = 0; u < NU; ++u) {
      const int i = lane + 64 * u;
#pragma unroll
      for (int j = 0; j + 1 < TAPS; ++j)
        if (j >= pad && i < len) h[(long)(j - pad) * channels + c0 + i] = win[u][j];
    }
  }
};

// sum_sp w[sp] acc[sp * stride + c] for a wave that owns columns [c0, c0 + 256) of n: w is lane
// sp's value (slices <= 64; a slice of weight 0 is not read).  VEC (n and stride multiples of 4,
// 16-byte aligned): several slices per pass, 16-byte loads; out(c, value) is called once per
// column by one lane.
template <bool VEC, typename F>
__device__ __forceinline__ void merge_slices(const float* __restrict__ acc, long stride, float w, int slices, int c0,
                                             int n, int lane, F out) {
  const int cols = min(256, n - c0);
  if constexpr (VEC) {
    const int pieces = cols / 4;
    int lpp = 1;
    while (lpp < pieces) lpp <<= 1;              // lanes per slice
    const int per = 64 / lpp, sub = lane / lpp, pc = lane & (lpp - 1);
    float v[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
    for (int s0 = 0; s0 < slices; s0 += per) {
      const int sp = s0 + sub;
      const float ws = __shfl(w, min(sp, 63));
      if (sp < slices && ws != 0.f && pc < pieces) {
        const float4 a = *reinterpret_cast<const float4*>(acc + sp * stride + c0 + 4 * pc);
        v[0] += ws * a.x;
        v[1] += ws * a.y;
        v[2] += ws * a.z;
        v[3] += ws * a.w;
      }
    }
    for (int off = lpp; off < 64; off <<= 1) {
#pragma unroll
      for (int k = 0; k < 4; ++k) v[k] += __shfl_xor(v[k], off);
    }
    if (sub == 0 && pc < pieces) {
#pragma unroll
      for (int k = 0; k < 4; ++k) out(c0 + 4 * pc + k, v[k]);
    }
  } else {
    for (int c = lane; c - lane < cols; c += 64) {
      float v = 0.f;
#pragma unroll 4
      for (int sp = 0; sp < slices; ++sp) {
        const float ws = __shfl(w, sp);
        if (c < cols && ws != 0.f) v += ws * acc[sp * stride + c0 + c];
      }
      if (c < cols) out(c0 + c, v);
    }
  }
}

// sum over a block of NT threads (NT multiple of 64, <= 1024); every thread gets it
template <int NT>
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = ft::wave_sum(v);
  constexpr int NW = NT / 64;
  if constexpr (NW == 1) return v;
  __syncthreads();   // red may still be read from a previous call
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int w = 0; w < NW; ++w) s += red[w];
  return s;
}

}  // namespace mx

#define MX_DISPATCH_T(bf16, ...)            \
  do {                                      \
    if (bf16) {                             \
      using T = ::mx::bf16_t;               \
      __VA_ARGS__;                          \
    } else {                                \
      using T = float;                      \
      __VA_ARGS__;                          \
    }                                       \
  } while (0)
