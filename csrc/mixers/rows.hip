// Row-wise kernels around an fp32 residual stream: embedding rows (optionally with a
// sinusoidal position vector), the fused "post-norm add + next pre-norm" step (also with a
// token shift of the normed row), the layer
// norm (weight and bias) that adds a sublayer's output to the residual, the tanh cap of
// the logits, per-head gated output norm (alone, or beside a second mixer's scaled rows), activations
// (relu^2, clamped / gelu / relu / silu GLU, gelu * token-side embedding) and the weighted row scatter-add
// that combines expert outputs.
#include <type_traits>

#include "mx_common.h"

namespace mx {

// out = table[id] * scale (+ a sinusoidal position vector when freqs is given: column 2i
// gets sin(p f_i), column 2i+1 cos(p f_i), with the angle p f_i formed in fp32)
template <typename T>
__global__ void embed_rows_kernel(float* __restrict__ out, const int* __restrict__ ids,
                                  const T* __restrict__ table, int width, int vocab, float scale,
                                  const int* __restrict__ positions, const float* __restrict__ freqs) {
  const int row = blockIdx.x;
  int id = ids[row];
  if (id < 0 || id >= vocab) id = 0;
  const float p = freqs != nullptr ? (float)positions[row] : 0.f;
  for (int i = threadIdx.x; i < width; i += blockDim.x) {
    float v = ld(table, (long)id * width + i) * scale;
    if (freqs != nullptr) {
      const float a = p * freqs[i >> 1];
      v += (i & 1) ? cosf(a) : sinf(a);
    }
    out[(long)row * width + i] = v;
  }
}

// a value of a row that is fp32 or bf16, decided at run time (uniform over the launch)
__device__ __forceinline__ float ldx(const void* p, int bf16, long i) {
  return bf16 ? ft::bf16_to_f32(((const bf16_t*)p)[i]) : ((const float*)p)[i];
}

// x (fp32 residual) = embed[cur] * scale + table[hash] per row (without `embed`: x +=
// table[hash]), hash = (prev * mul_prev + cur * mul_cur) mod
// buckets with prev the token before the row's own in its sequence: the row above within a
// segment, last_tok[slot] for a segment's first row (pos0 > 0), and for a sequence's first
// token row `buckets` instead.  One workgroup per row; pair_last_kernel stores each
// segment's last token afterwards (a second launch: another row of the segment may still
// be reading the old one).
template <typename T>
__global__ void pair_embed_add_kernel(float* __restrict__ x, const int* __restrict__ ids,
                                      const T* __restrict__ table, int width, long mul_prev, long mul_cur,
                                      int buckets, const int* __restrict__ start, const int* __restrict__ pos0,
                                      const int* __restrict__ slot, int num_segs, const int* __restrict__ last_tok,
                                      int num_slots, const T* __restrict__ embed, int vocab, float scale) {
  const int row = blockIdx.x;
  if (embed != nullptr) {                 // every row gets its embedding row, padding rows too
    int id = ids[row];
    if (id < 0 || id >= vocab) id = 0;
    for (int i = threadIdx.x; i < width; i += blockDim.x)
      x[(long)row * width + i] = ld(embed, (long)id * width + i) * scale;
  }
  if (row >= start[num_segs]) return;
  int lo_s = 0, hi_s = num_segs;
  while (hi_s - lo_s > 1) {
    const int mid = (lo_s + hi_s) >> 1;
    if (start[mid] <= row) lo_s = mid; else hi_s = mid;
  }
  const int sg = lo_s;
  const int sl = slot[sg];
  if (sl < 0 || sl >= num_slots) return;
  long prev;
  if (row > start[sg]) prev = ids[row - 1];
  else prev = pos0[sg] > 0 ? last_tok[sl] : -1;
  long idx = buckets;
  if (prev >= 0) {
    idx = (prev * mul_prev + (long)ids[row] * mul_cur) % buckets;
    if (idx < 0) idx += buckets;
  }
  for (int i = threadIdx.x; i < width; i += blockDim.x) x[(long)row * width + i] += ld(table, idx * width + i);
}

__global__ void pair_last_kernel(const int* __restrict__ ids, const int* __restrict__ start,
                                 const int* __restrict__ slot, int num_segs, int* __restrict__ last_tok,
                                 int num_slots) {
  const int sg = blockIdx.x * blockDim.x + threadIdx.x;
  if (sg >= num_segs) return;
  const int sl = slot[sg];
  const int a = start[sg], b = start[sg + 1];
  if (sl < 0 || sl >= num_slots || b <= a) return;
  last_tok[sl] = ids[b - 1];
}

// residual (fp32, in place): x += mult * (y1 + y2);  out = rms_norm(x) * next_w (TO).
// y1 / y2 are fp32 or bf16 each and optional, as is out.
template <typename TO, int NT>
__global__ void add_scaled_rms_norm_kernel(float* __restrict__ x, const void* __restrict__ y1, int y1_bf16,
                                           long y1_stride, const void* __restrict__ y2, int y2_bf16,
                                           long y2_stride, float mult, const float* __restrict__ next_w,
                                           TO* __restrict__ out, int width, float eps) {
  __shared__ float red[NT / 64];
  const long row = blockIdx.x;
  float* xr = x + row * width;
  float ss = 0.f;
  for (int i = threadIdx.x; i < width; i += NT) {
    float v = xr[i];
    if (y1 != nullptr) {
      float y = ldx(y1, y1_bf16, row * y1_stride + i);
      if (y2 != nullptr) y += ldx(y2, y2_bf16, row * y2_stride + i);
      v += mult * y;
      xr[i] = v;
    }
    ss += v * v;
  }
  if (out == nullptr) return;
  ss = block_sum<NT>(ss, red);
  const float r = 1.0f / sqrtf(ss / (float)width + eps);
  // each thread re-reads only what it wrote itself
  for (int i = threadIdx.x; i < width; i += NT) st(out, row * width + i, xr[i] * r * next_w[i]);
}

// out (fp32) = scale * (a / rms(a) * wa + b / rms(b) * wb), one workgroup per row
template <typename T, int NT>
__global__ void dual_rms_mean_kernel(float* __restrict__ out, const T* __restrict__ a, long a_stride,
                                     const T* __restrict__ b, long b_stride, const float* __restrict__ wa,
                                     const float* __restrict__ wb, int width, float eps, float scale) {
  __shared__ float red[NT / 64];
  const long row = blockIdx.x;
  const T* ar = a + row * a_stride;
  const T* br = b + row * b_stride;
  float sa = 0.f, sb = 0.f;
  for (int i = threadIdx.x; i < width; i += NT) {
    const float u = ld(ar, i), v = ld(br, i);
    sa += u * u;
    sb += v * v;
  }
  sa = block_sum<NT>(sa, red);
  sb = block_sum<NT>(sb, red);
  const float ra = 1.0f / sqrtf(sa / (float)width + eps), rb = 1.0f / sqrtf(sb / (float)width + eps);
  for (int i = threadIdx.x; i < width; i += NT)
    out[row * width + i] = scale * (ld(ar, i) * ra * wa[i] + ld(br, i) * rb * wb[i]);
}

// out = o * sigmoid(g), o fp32 dense rows, g rows g_stride apart
template <typename TG, typename TO>
__global__ void sigmoid_gate_kernel(TO* __restrict__ out, const float* __restrict__ o, const TG* __restrict__ g,
                                    long g_stride, long rows, int n) {
  const long total = rows * n;
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (long)gridDim.x * blockDim.x) {
    const long r = i / n;
    const int c = (int)(i % n);
    st(out, i, o[i] * sigmoidf_(ld(g, r * g_stride + c)));
  }
}

// layer norm with weight and bias, ln(u) = (u - mean) / sqrt(var + eps) * w + b with var
// the mean squared deviation (two passes), around an fp32 residual x:
//   y given:            x += ln(y);  cast = x
//   y null, out null:   x  = ln(x);  cast = x
//   y null, out given:  out = ln(x)  (x untouched)
template <typename TY, typename TO, int NT>
__global__ void layer_norm_kernel(float* __restrict__ x, const TY* __restrict__ y, long y_stride,
                                  const float* __restrict__ w, const float* __restrict__ b,
                                  TO* __restrict__ out, TO* __restrict__ cast, int width, float eps) {
  __shared__ float red[NT / 64];
  const long row = blockIdx.x;
  float* xr = x + row * width;
  const TY* yr = y != nullptr ? y + row * y_stride : nullptr;
  auto src = [&](int i) { return yr != nullptr ? ld(yr, i) : xr[i]; };
  float sum = 0.f;
  for (int i = threadIdx.x; i < width; i += NT) sum += src(i);
  const float mean = block_sum<NT>(sum, red) / (float)width;
  float ss = 0.f;
  for (int i = threadIdx.x; i < width; i += NT) {
    const float d = src(i) - mean;
    ss += d * d;
  }
  const float r = 1.0f / sqrtf(block_sum<NT>(ss, red) / (float)width + eps);
  for (int i = threadIdx.x; i < width; i += NT) {
    const float v = (src(i) - mean) * r * w[i] + b[i];
    if (out != nullptr) {
      st(out, row * width + i, v);
    } else {
      const float nx = yr != nullptr ? xr[i] + v : v;
      xr[i] = nx;
      if (cast != nullptr) st(cast, row * width + i, nx);
    }
  }
}

// x <- cap * tanh(x / cap); infinite entries stay
__global__ void tanh_cap_kernel(float* __restrict__ x, long n, float cap) {
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long)gridDim.x * blockDim.x) {
    const float v = x[i];
    if (isfinite(v)) x[i] = cap * tanhf(v / cap);
  }
}

// A row of a workgroup in registers: 4 C entries per thread, four neighbours at a time (16-byte
// fp32 or 8-byte bf16 accesses when `vec`), width <= 4 C NT.
template <typename T, int NT, int C>
__device__ __forceinline__ void load_row(float (&v)[C][4], const T* p, int width, int vec) {
#pragma unroll
  for (int c = 0; c < C; ++c) {
    const int i = (c * NT + threadIdx.x) * 4;
    if (vec && i < width) {
      if constexpr (sizeof(T) == 2) {
        const uint2 u = *reinterpret_cast<const uint2*>(p + i);
        ft::unpack2(u.x, v[c][0], v[c][1]);
        ft::unpack2(u.y, v[c][2], v[c][3]);
      } else {
        const float4 u = *reinterpret_cast<const float4*>(p + i);
        v[c][0] = u.x; v[c][1] = u.y; v[c][2] = u.z; v[c][3] = u.w;
      }
    } else {
#pragma unroll
      for (int k = 0; k < 4; ++k) v[c][k] = i + k < width ? ld(p, i + k) : 0.f;
    }
  }
}

template <typename T, int NT, int C>
__device__ __forceinline__ void store_row(T* p, const float (&v)[C][4], int width, int vec) {
#pragma unroll
  for (int c = 0; c < C; ++c) {
    const int i = (c * NT + threadIdx.x) * 4;
    if (vec && i < width) {
      if constexpr (sizeof(T) == 2) {
        *reinterpret_cast<uint2*>(p + i) = make_uint2(ft::pack2(v[c][0], v[c][1]), ft::pack2(v[c][2], v[c][3]));
      } else {
        *reinterpret_cast<float4*>(p + i) = make_float4(v[c][0], v[c][1], v[c][2], v[c][3]);
      }
    } else {
#pragma unroll
      for (int k = 0; k < 4; ++k)
        if (i + k < width) st(p, i + k, v[c][k]);
    }
  }
}

// sums of two values over a block; every thread gets both
template <int NT>
__device__ __forceinline__ void block_sum2(float& a, float& b, float (*red)[2]) {
  a = ft::wave_sum(a);
  b = ft::wave_sum(b);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) {
    red[threadIdx.x >> 6][0] = a;
    red[threadIdx.x >> 6][1] = b;
  }
  __syncthreads();
  a = b = 0.f;
#pragma unroll
  for (int w = 0; w < NT / 64; ++w) {
    a += red[w][0];
    b += red[w][1];
  }
}

template <int C>
__device__ __forceinline__ float sum_sq(const float (&v)[C][4]) {
  float s = 0.f;
#pragma unroll
  for (int c = 0; c < C; ++c)
#pragma unroll
    for (int k = 0; k < 4; ++k) s += v[c][k] * v[c][k];
  return s;
}

// residual (fp32, in place): x += rms_norm(y) * wb (y as it is without wb) (+ add_vec);
// out = rms_norm(x) * next_w (TO);  cast = x (TO).  Every part is optional.
template <typename TY, typename TO, int NT, int C>
__global__ void __launch_bounds__(NT)
add_rms_norm_kernel(float* __restrict__ x, const TY* __restrict__ y, long y_stride, const float* __restrict__ wb,
                    const float* __restrict__ add_vec, const float* __restrict__ next_w, TO* __restrict__ out,
                    TO* __restrict__ cast, int width, float eps, int vec) {
  __shared__ float red[NT / 64];
  const long row = blockIdx.x;
  float v[C][4], t[C][4], w[C][4];
  load_row<float, NT, C>(v, x + row * width, width, vec);
  if (y != nullptr) {
    load_row<TY, NT, C>(t, y + row * y_stride, width, vec);
    if (wb != nullptr) {
      load_row<float, NT, C>(w, wb, width, vec);
      const float r = 1.0f / sqrtf(block_sum<NT>(sum_sq<C>(t), red) / (float)width + eps);
#pragma unroll
      for (int c = 0; c < C; ++c)
#pragma unroll
        for (int k = 0; k < 4; ++k) t[c][k] *= r * w[c][k];
    }
#pragma unroll
    for (int c = 0; c < C; ++c)
#pragma unroll
      for (int k = 0; k < 4; ++k) v[c][k] += t[c][k];
  }
  if (add_vec != nullptr) {
    load_row<float, NT, C>(w, add_vec, width, vec);
#pragma unroll
    for (int c = 0; c < C; ++c)
#pragma unroll
      for (int k = 0; k < 4; ++k) v[c][k] += w[c][k];
  }
  if (y != nullptr || add_vec != nullptr) store_row<float, NT, C>(x + row * width, v, width, vec);
  if (cast != nullptr) store_row<TO, NT, C>(cast + row * width, v, width, vec);
  if (out != nullptr) {
    load_row<float, NT, C>(w, next_w, width, vec);
    const float r = 1.0f / sqrtf(block_sum<NT>(sum_sq<C>(v), red) / (float)width + eps);
#pragma unroll
    for (int c = 0; c < C; ++c)
#pragma unroll
      for (int k = 0; k < 4; ++k) v[c][k] *= r * w[c][k];
    store_row<TO, NT, C>(out + row * width, v, width, vec);
  }
}

// ---------------------------------------------------------------------------------
// the step between layers with a token shift, one workgroup per row:
//   x_out = x_in + rms_norm(y) * wb (without y: x_out = x_in, not written)
//   h = rms_norm(x_out) * w;  out = h + (h' - h) * shift
// with h' the h of the token before: of the row above within a segment (recomputed here from
// that row's x_in and y, so x_out must be another buffer than x_in when a segment has several
// rows), of the state slot for a segment's first row, zeros for a sequence's first token.  A
// one-row segment also leaves its h in the slot; shift_state_kernel does that for longer ones
// afterwards (a slot may still be read by the segment's first row here).
// ---------------------------------------------------------------------------------
template <typename TY, typename TO, int NT, int C>
__global__ void __launch_bounds__(NT)
add_norm_shift_kernel(float* x_out, const float* x_in, const TY* __restrict__ y, long y_stride,
                      const float* __restrict__ wb, const float* __restrict__ w, const float* __restrict__ shift,
                      TO* __restrict__ out, float* state, int num_slots, const int* __restrict__ start,
                      const int* __restrict__ pos0, const int* __restrict__ slot, int num_segs, int width,
                      float eps, int vec) {
  __shared__ float red[NT / 64][2];
  const long row = blockIdx.x;
  int sl = -1, rel = 0, n = 1;
  bool old = false;
  if (row < start[num_segs]) {
    const int sg = segment_of(start, num_segs, (int)row);
    rel = (int)row - start[sg];
    n = start[sg + 1] - start[sg];
    sl = slot[sg];
    if (sl >= num_slots) sl = -1;
    old = sl >= 0 && pos0[sg] > 0;
  }
  float xa[C][4], xp[C][4], t[C][4];
  load_row<float, NT, C>(xa, x_in + row * width, width, vec);
  if (rel > 0) load_row<float, NT, C>(xp, x_in + (row - 1) * width, width, vec);
  if (y != nullptr) {
    float yp[C][4];
    load_row<TY, NT, C>(t, y + row * y_stride, width, vec);
    if (rel > 0) load_row<TY, NT, C>(yp, y + (row - 1) * y_stride, width, vec);
    float sa = sum_sq<C>(t), sb = rel > 0 ? sum_sq<C>(yp) : 0.f;
    block_sum2<NT>(sa, sb, red);
    const float ra = 1.0f / sqrtf(sa / (float)width + eps), rb = 1.0f / sqrtf(sb / (float)width + eps);
    float wv[C][4];
    load_row<float, NT, C>(wv, wb, width, vec);
#pragma unroll
    for (int c = 0; c < C; ++c)
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        xa[c][k] += t[c][k] * ra * wv[c][k];
        if (rel > 0) xp[c][k] += yp[c][k] * rb * wv[c][k];
      }
    store_row<float, NT, C>(x_out + row * width, xa, width, vec);
  }
  float sa = sum_sq<C>(xa), sb = rel > 0 ? sum_sq<C>(xp) : 0.f;
  block_sum2<NT>(sa, sb, red);
  const float ra = 1.0f / sqrtf(sa / (float)width + eps), rb = 1.0f / sqrtf(sb / (float)width + eps);
  load_row<float, NT, C>(t, w, width, vec);
#pragma unroll
  for (int c = 0; c < C; ++c)
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      xa[c][k] *= ra * t[c][k];
      xp[c][k] = rel > 0 ? xp[c][k] * (rb * t[c][k]) : 0.f;
    }
  if (rel == 0 && old) load_row<float, NT, C>(xp, state + (long)sl * width, width, vec);
  if (sl >= 0 && n == 1) store_row<float, NT, C>(state + (long)sl * width, xa, width, vec);
  load_row<float, NT, C>(t, shift, width, vec);
#pragma unroll
  for (int c = 0; c < C; ++c)
#pragma unroll
    for (int k = 0; k < 4; ++k) xa[c][k] += (xp[c][k] - xa[c][k]) * t[c][k];
  store_row<TO, NT, C>(out + row * width, xa, width, vec);
}

// the h of each longer segment's last row, from its x, into the segment's slot; grid segments
template <int NT, int C>
__global__ void __launch_bounds__(NT)
shift_state_kernel(float* __restrict__ state, int num_slots, const float* __restrict__ x, const float* __restrict__ w,
                   const int* __restrict__ start, const int* __restrict__ slot, int width, float eps, int vec) {
  __shared__ float red[NT / 64][2];
  const int s = blockIdx.x;
  const int n = start[s + 1] - start[s], sl = slot[s];
  if (n < 2 || sl < 0 || sl >= num_slots) return;
  float xa[C][4], t[C][4];
  load_row<float, NT, C>(xa, x + (long)(start[s + 1] - 1) * width, width, vec);
  float sa = sum_sq<C>(xa), sb = 0.f;
  block_sum2<NT>(sa, sb, red);
  const float ra = 1.0f / sqrtf(sa / (float)width + eps);
  load_row<float, NT, C>(t, w, width, vec);
#pragma unroll
  for (int c = 0; c < C; ++c)
#pragma unroll
    for (int k = 0; k < 4; ++k) xa[c][k] *= ra * t[c][k];
  store_row<float, NT, C>(state + (long)sl * width, xa, width, vec);
}

// one wave per (row, head): out = o / rms(o) * w * sigmoid(gate), or * silu(gate)
template <typename TG, typename TO>
__global__ void head_rms_gate_kernel(TO* __restrict__ out, const float* __restrict__ o,
                                     const float* __restrict__ w, const TG* __restrict__ gate,
                                     long gate_stride, long pairs, int heads, int dv, float eps, int silu) {
  const long pair = (long)blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (pair >= pairs) return;
  const int lane = threadIdx.x & 63;
  const long row = pair / heads;
  const int h = (int)(pair % heads);
  const float* op = o + (row * heads + h) * dv;
  float ss = 0.f;
  for (int i = lane; i < dv; i += 64) ss += op[i] * op[i];
  ss = ft::wave_sum(ss);
  const float r = 1.0f / sqrtf(ss / (float)dv + eps);
  for (int i = lane; i < dv; i += 64) {
    const float gp = ld(gate, row * gate_stride + (long)h * dv + i);
    const float g = silu ? gp * sigmoidf_(gp) : sigmoidf_(gp);
    st(out, (row * heads + h) * dv + i, op[i] * r * w[i] * g);
  }
}

// rows [a_scale * a (n) | o_scale * o / rms(o) per head * silu(gate)]: one wave per (row, item),
// items are the heads of o, then pieces of 256 columns of a
template <typename T>
__global__ void scaled_pair_rows_kernel(T* __restrict__ out, const float* __restrict__ a, int n, float a_scale,
                                        const float* __restrict__ o, const T* __restrict__ gate, long gate_stride,
                                        float o_scale, long waves, int items, int heads, int dv, float eps) {
  const long w = (long)blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (w >= waves) return;
  const int lane = threadIdx.x & 63;
  const long row = w / items;
  const int it = (int)(w % items);
  T* orow = out + row * (n + (long)heads * dv);
  if (it >= heads) {
    const int c0 = (it - heads) * 256;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int c = c0 + lane + 64 * u;
      if (c < n) st(orow, c, a[row * n + c] * a_scale);
    }
    return;
  }
  const float* op = o + (row * heads + it) * dv;
  float ss = 0.f;
  for (int i = lane; i < dv; i += 64) ss += op[i] * op[i];
  const float r = 1.0f / sqrtf(ft::wave_sum(ss) / (float)dv + eps) * o_scale;
  for (int i = lane; i < dv; i += 64) {
    const float g = ld(gate, row * gate_stride + (long)it * dv + i);
    st(orow, n + (long)it * dv + i, op[i] * r * (g * sigmoidf_(g)));
  }
}

template <typename T>
__global__ void relu_sq_kernel(T* __restrict__ x, long n) {
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long)gridDim.x * blockDim.x) {
    const float v = fmaxf(ld(x, i), 0.f);
    st(x, i, v * v);
  }
}

// out[r, c] = relu(u[r, c])^2 for the first ff columns of wider rows
template <typename T>
__global__ void relu_sq_rows_kernel(T* __restrict__ out, const T* __restrict__ u, long u_stride, long rows, int ff) {
  const long n = rows * ff;
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long)gridDim.x * blockDim.x) {
    const float v = fmaxf(ld(u, (i / ff) * u_stride + i % ff), 0.f);
    st(out, i, v * v);
  }
}

// out[row] += sum_k w[row, k] * y[idx[row, k]]: combines the outputs of the experts each
// row chose, y being in another row order (sorted by expert).  grid rows.
template <typename TY>
__global__ void gather_add_rows_kernel(float* __restrict__ out, const TY* __restrict__ y,
                                       const int* __restrict__ idx, const float* __restrict__ w, int top,
                                       int width, long y_rows) {
  const long row = blockIdx.x;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    float acc = 0.f;
    for (int k = 0; k < top; ++k) {
      const long src = idx[row * top + k];
      if (src >= 0 && src < y_rows) acc += w[row * top + k] * ld(y, src * width + c);
    }
    out[row * width + c] += acc;
  }
}

// Gated linear units on rows [gate (ff) | up (ff) | ...], activation by a functor; VEC: eight
// neighbouring bf16 (four fp32) entries per thread, 16-byte accesses
template <typename T> struct GluVec;
template <> struct GluVec<float> { static constexpr int N = 4; };
template <> struct GluVec<bf16_t> { static constexpr int N = 8; };

__device__ __forceinline__ void load16(const float* p, float (&v)[4]) {
  const float4 u = *reinterpret_cast<const float4*>(p);
  v[0] = u.x; v[1] = u.y; v[2] = u.z; v[3] = u.w;
}
__device__ __forceinline__ void load16(const bf16_t* p, float (&v)[8]) { ft::load8(*reinterpret_cast<const uint4*>(p), v); }
__device__ __forceinline__ void store16(float* p, const float (&v)[4]) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}
__device__ __forceinline__ void store16(bf16_t* p, const float (&v)[8]) {
  *reinterpret_cast<uint4*>(p) =
      make_uint4(ft::pack2(v[0], v[1]), ft::pack2(v[2], v[3]), ft::pack2(v[4], v[5]), ft::pack2(v[6], v[7]));
}

template <typename T, typename F>
__device__ __forceinline__ void glu_rows(T* __restrict__ out, const T* __restrict__ gu, long gu_stride, long rows, int ff,
                                         int vec, F act) {
  constexpr int N = GluVec<T>::N;
  const long step = (long)gridDim.x * blockDim.x, i0 = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (vec) {
    const int per = ff / N;
    for (long i = i0; i < rows * per; i += step) {
      const long r = i / per;
      const int c = (int)(i - r * per) * N;
      float g[N], u[N];
      load16(gu + r * gu_stride + c, g);
      load16(gu + r * gu_stride + ff + c, u);
#pragma unroll
      for (int k = 0; k < N; ++k) g[k] = act(g[k], u[k]);
      store16(out + r * ff + c, g);
    }
    return;
  }
  for (long i = i0; i < rows * ff; i += step) {
    const long r = i / ff;
    const int c = (int)(i % ff);
    st(out, i, act(ld(gu, r * gu_stride + c), ld(gu, r * gu_stride + ff + c)));
  }
}

// rows [gate (ff) | up (ff) | ...]: g = min(gate, limit), u = clamp(up, +-limit),
// out = g * sigmoid(1.702 g) * (u + 1)
template <typename T>
__global__ void clamp_swiglu_kernel(T* __restrict__ out, const T* __restrict__ gu, long gu_stride,
                                    long rows, int ff, float limit, int vec) {
  glu_rows(out, gu, gu_stride, rows, ff, vec, [=](float g, float u) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g * sigmoidf_(1.702f * g) * (u + 1.0f);
  });
}

__device__ __forceinline__ float gelu_tanh_(float z) {
  return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// rows [gate (ff) | up (ff)]: out = act(gate) * up, act = gelu_tanh (0), relu (1) or silu (2)
template <typename T>
__global__ void act_glu_kernel(T* __restrict__ out, const T* __restrict__ gu, long gu_stride, long rows, int ff,
                               int act, int vec) {
  glu_rows(out, gu, gu_stride, rows, ff, vec, [=](float g, float u) {
    return (act == 2 ? g * sigmoidf_(g) : act == 1 ? fmaxf(g, 0.f) : gelu_tanh_(g)) * u;
  });
}

template <typename T>
__global__ void side_gate_kernel(T* __restrict__ out, const T* __restrict__ gpre,
                                 const T* __restrict__ table, long table_stride,
                                 const int* __restrict__ ids, int col0, long rows, int sd, int vocab) {
  const long n = rows * sd;
  for (long i = (long)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (long)gridDim.x * blockDim.x) {
    const long r = i / sd;
    const int c = (int)(i % sd);
    int id = ids[r];
    if (id < 0 || id >= vocab) id = 0;
    st(out, i, gelu_tanh_(ld(gpre, i)) * ld(table, (long)id * table_stride + col0 + c));
  }
}

// out[rows[i]] += w_i * y[i]; rows == nullptr: identity.  No row repeats within a call.
template <typename TY, typename TW>
__global__ void scale_add_rows_kernel(float* __restrict__ out, const TY* __restrict__ y,
                                      const int* __restrict__ rows, const TW* __restrict__ weights,
                                      int sigmoid, int width, int out_rows) {
  const long i = blockIdx.x;
  const long dst = rows != nullptr ? rows[i] : i;
  if (dst < 0 || dst >= out_rows) return;
  float w = ld(weights, i);
  if (sigmoid) w = sigmoidf_(w);
  for (int c = threadIdx.x; c < width; c += blockDim.x)
    out[dst * width + c] += w * ld(y, i * width + c);
}

}  // namespace mx

using namespace mx;

extern "C" int mx_embed_rows(float* out, const int* ids, const void* table, int bf16, int rows,
                             int width, int vocab, float scale, const int* positions, const float* freqs,
                             hipStream_t s) {
  if (rows <= 0) return 0;
  if (freqs != nullptr && positions == nullptr) return -1;
  MX_DISPATCH_T(bf16, hipLaunchKernelGGL((embed_rows_kernel<T>), dim3(rows), dim3(256), 0, s, out, ids,
                                         (const T*)table, width, vocab, scale, positions, freqs));
  return (int)hipGetLastError();
}

template <typename TY, typename TO>
static void launch_layer_norm(float* x, const void* y, long ys, const float* w, const float* b, void* out,
                              void* cast, int rows, int width, float eps, hipStream_t s) {
  hipLaunchKernelGGL((layer_norm_kernel<TY, TO, 256>), dim3(rows), dim3(256), 0, s, x, (const TY*)y, ys, w, b,
                     (TO*)out, (TO*)cast, width, eps);
}

extern "C" int mx_layer_norm(float* x, const void* y, int y_bf16, long y_stride, const float* w, const float* b,
                             void* out, void* cast, int out_bf16, int rows, int width, float eps, hipStream_t s) {
  if (rows <= 0) return 0;
  if (y != nullptr && out != nullptr) return -1;
  if (y_bf16) {
    if (out_bf16) launch_layer_norm<bf16_t, bf16_t>(x, y, y_stride, w, b, out, cast, rows, width, eps, s);
    else launch_layer_norm<bf16_t, float>(x, y, y_stride, w, b, out, cast, rows, width, eps, s);
  } else {
    if (out_bf16) launch_layer_norm<float, bf16_t>(x, y, y_stride, w, b, out, cast, rows, width, eps, s);
    else launch_layer_norm<float, float>(x, y, y_stride, w, b, out, cast, rows, width, eps, s);
  }
  return (int)hipGetLastError();
}

constexpr int kRowThreads = 512;
constexpr int kRowMaxWidth = kRowThreads * 4 * 8;

// calls f with the number of register chunks a row of this width takes, as a constant
template <typename F>
static void row_chunks(int width, F f) {
  const int chunks = (width + kRowThreads * 4 - 1) / (kRowThreads * 4);
  if (chunks <= 1) f(std::integral_constant<int, 1>{});
  else if (chunks <= 2) f(std::integral_constant<int, 2>{});
  else if (chunks <= 4) f(std::integral_constant<int, 4>{});
  else f(std::integral_constant<int, 8>{});
}

template <typename TY, typename TO>
static void launch_add_rms(float* x, const void* y, long ys, const float* wb, const float* av,
                           const float* nw, void* out, void* cast, int rows, int width, float eps,
                           hipStream_t s) {
  const int vec = width % 4 == 0 && (y == nullptr || (ys % 4 == 0 && ((uintptr_t)y) % (4 * sizeof(TY)) == 0)) &&
                  ((uintptr_t)x | (uintptr_t)wb | (uintptr_t)av | (uintptr_t)nw) % 16 == 0 &&
                  ((uintptr_t)out | (uintptr_t)cast) % (4 * sizeof(TO)) == 0;
  row_chunks(width, [&](auto c) {
    hipLaunchKernelGGL((add_rms_norm_kernel<TY, TO, kRowThreads, decltype(c)::value>), dim3(rows), dim3(kRowThreads), 0,
                       s, x, (const TY*)y, ys, wb, av, nw, (TO*)out, (TO*)cast, width, eps, vec);
  });
}

extern "C" int mx_add_rms_norm(float* x, const void* y, int y_bf16, long y_stride, const float* wb,
                               const float* add_vec, const float* next_w, void* out, void* cast,
                               int out_bf16, int rows, int width, float eps, hipStream_t s) {
  if (rows <= 0) return 0;
  if (width < 1 || width > kRowMaxWidth) return -1;
  if (y_bf16) {
    if (out_bf16) launch_add_rms<bf16_t, bf16_t>(x, y, y_stride, wb, add_vec, next_w, out, cast, rows, width, eps, s);
    else launch_add_rms<bf16_t, float>(x, y, y_stride, wb, add_vec, next_w, out, cast, rows, width, eps, s);
  } else {
    if (out_bf16) launch_add_rms<float, bf16_t>(x, y, y_stride, wb, add_vec, next_w, out, cast, rows, width, eps, s);
    else launch_add_rms<float, float>(x, y, y_stride, wb, add_vec, next_w, out, cast, rows, width, eps, s);
  }
  return (int)hipGetLastError();
}

extern "C" int mx_head_rms_gate(void* out, int out_bf16, const float* o, const float* w,
                                const void* gate, int gate_bf16, long gate_stride, long rows, int heads,
                                int dv, float eps, int silu, hipStream_t s) {
  const long pairs = rows * heads;
  if (pairs <= 0) return 0;
  const dim3 grid((unsigned)((pairs + 3) / 4)), block(256);
  if (gate_bf16 && out_bf16)
    hipLaunchKernelGGL((head_rms_gate_kernel<bf16_t, bf16_t>), grid, block, 0, s, (bf16_t*)out, o, w,
                       (const bf16_t*)gate, gate_stride, pairs, heads, dv, eps, silu);
  else if (!gate_bf16 && !out_bf16)
    hipLaunchKernelGGL((head_rms_gate_kernel<float, float>), grid, block, 0, s, (float*)out, o, w,
                       (const float*)gate, gate_stride, pairs, heads, dv, eps, silu);
  else
    return -1;
  return (int)hipGetLastError();
}

extern "C" int mx_scaled_pair_rows(void* out, int bf16, const float* a, int n, float a_scale, const float* o,
                                   const void* gate, long gate_stride, float o_scale, long rows, int heads, int dv,
                                   float eps, hipStream_t s) {
  const int items = heads + (n + 255) / 256;
  const long waves = rows * items;
  if (waves <= 0) return 0;
  const dim3 grid((unsigned)((waves + 3) / 4)), block(256);
  MX_DISPATCH_T(bf16, hipLaunchKernelGGL((scaled_pair_rows_kernel<T>), grid, block, 0, s, (T*)out, a, n, a_scale, o,
                                         (const T*)gate, gate_stride, o_scale, waves, items, heads, dv, eps));
  return (int)hipGetLastError();
}

static inline unsigned ew_grid(long n) {
  long g = (n + 255) / 256;
  return (unsigned)(g < 1 ? 1 : g > 65535 ? 65535 : g);
}

// whole 16-byte pieces in every row of gate, up and out
static inline int glu_vec(const void* out, const void* gu, int bf16, long gu_stride, int ff) {
  const int n = bf16 ? 8 : 4;
  return ff % n == 0 && gu_stride % n == 0 && ((uintptr_t)out | (uintptr_t)gu) % 16 == 0;
}

extern "C" int mx_tanh_cap(float* x, long n, float cap, hipStream_t s) {
  if (n <= 0) return 0;
  if (!(cap > 0.f)) return -1;
  hipLaunchKernelGGL(tanh_cap_kernel, dim3(ew_grid(n)), dim3(256), 0, s, x, n, cap);
  return (int)hipGetLastError();
}

extern "C" int mx_relu_sq(void* x, int bf16, long n, hipStream_t s) {
  if (n <= 0) return 0;
  MX_DISPATCH_T(bf16, hipLaunchKernelGGL((relu_sq_kernel<T>), dim3(ew_grid(n)), dim3(256), 0, s, (T*)x, n));
  return (int)hipGetLastError();
}

extern "C" int mx_relu_sq_rows(void* out, const void* u, int bf16, long u_stride, long rows, int ff, hipStream_t s) {
  if (rows * ff <= 0) return 0;
  MX_DISPATCH_T(bf16, hipLaunchKernelGGL((relu_sq_rows_kernel<T>), dim3(ew_grid(rows * ff)), dim3(256), 0, s,
                                         (T*)out, (const T*)u, u_stride, rows, ff));
  return (int)hipGetLastError();
}

extern "C" int mx_gather_add_rows(float* out, const void* y, int y_bf16, const int* idx, const float* w, long rows,
                                  int top, int width, long y_rows, hipStream_t s) {
  if (rows <= 0 || top <= 0) return 0;
  if (rows > 0x7fffffffL) return -1;
  MX_DISPATCH_T(y_bf16, hipLaunchKernelGGL((gather_add_rows_kernel<T>), dim3((unsigned)rows), dim3(256), 0, s, out,
                                           (const T*)y, idx, w, top, width, y_rows));
  return (int)hipGetLastError();
}

extern "C" int mx_clamp_swiglu(void* out, const void* gu, int bf16, long gu_stride, long rows, int ff,
                               float limit, hipStream_t s) {
  if (rows * ff <= 0) return 0;
  const int vec = glu_vec(out, gu, bf16, gu_stride, ff);
  MX_DISPATCH_T(bf16, hipLaunchKernelGGL((clamp_swiglu_kernel<T>), dim3(ew_grid(vec ? rows * (ff / GluVec<T>::N) : rows * ff)),
                                         dim3(256), 0, s, (T*)out, (const T*)gu, gu_stride, rows, ff, limit, vec));
  return (int)hipGetLastError();
}

extern "C" int mx_act_glu(void* out, const void* gu, int bf16, long gu_stride, long rows, int ff, int act,
                          hipStream_t s) {
  if (rows * ff <= 0) return 0;
  if (act < 0 || act > 2) return -1;
  const int vec = glu_vec(out, gu, bf16, gu_stride, ff);
  MX_DISPATCH_T(bf16, hipLaunchKernelGGL((act_glu_kernel<T>), dim3(ew_grid(vec ? rows * (ff / GluVec<T>::N) : rows * ff)),
                                         dim3(256), 0, s, (T*)out, (const T*)gu, gu_stride, rows, ff, act, vec));
  return (int)hipGetLastError();
}

extern "C" int mx_side_gate(void* out, const void* gpre, const void* table, int bf16, long table_stride,
                            const int* ids, int col0, long rows, int sd, int vocab, hipStream_t s) {
  if (rows * sd <= 0) return 0;
  MX_DISPATCH_T(bf16, hipLaunchKernelGGL((side_gate_kernel<T>), dim3(ew_grid(rows * sd)), dim3(256), 0, s,
                                         (T*)out, (const T*)gpre, (const T*)table, table_stride, ids, col0,
                                         rows, sd, vocab));
  return (int)hipGetLastError();
}

extern "C" int mx_scale_add_rows(float* out, const void* y, int y_bf16, const int* rows,
                                 const void* weights, int w_bf16, int sigmoid, long n, int width,
                                 int out_rows, hipStream_t s) {
  if (n <= 0) return 0;
  const dim3 grid((unsigned)n), block(256);
  if (y_bf16 && w_bf16)
    hipLaunchKernelGGL((scale_add_rows_kernel<bf16_t, bf16_t>), grid, block, 0, s, out, (const bf16_t*)y,
                       rows, (const bf16_t*)weights, sigmoid, width, out_rows);
  else if (y_bf16)
    hipLaunchKernelGGL((scale_add_rows_kernel<bf16_t, float>), grid, block, 0, s, out, (const bf16_t*)y,
                       rows, (const float*)weights, sigmoid, width, out_rows);
  else if (w_bf16)
    return -1;
  else
    hipLaunchKernelGGL((scale_add_rows_kernel<float, float>), grid, block, 0, s, out, (const float*)y,
                       rows, (const float*)weights, sigmoid, width, out_rows);
  return (int)hipGetLastError();
}

extern "C" int mx_pair_embed_add(float* x, const int* ids, const void* table, int bf16, int rows, int width,
                                 long mul_prev, long mul_cur, int buckets, const int* start, const int* pos0,
                                 const int* slot, int num_segs, int* last_tok, int num_slots, const void* embed,
                                 int vocab, float scale, hipStream_t s) {
  if (rows <= 0 || num_segs <= 0) return 0;
  if (buckets < 1 || width < 1) return -1;
  MX_DISPATCH_T(bf16, hipLaunchKernelGGL((pair_embed_add_kernel<T>), dim3(rows), dim3(256), 0, s, x, ids,
                                         (const T*)table, width, mul_prev, mul_cur, buckets, start, pos0, slot,
                                         num_segs, last_tok, num_slots, (const T*)embed, vocab, scale));
  hipLaunchKernelGGL(pair_last_kernel, dim3((num_segs + 63) / 64), dim3(64), 0, s, ids, start, slot, num_segs, last_tok,
                     num_slots);
  return (int)hipGetLastError();
}

extern "C" int mx_add_scaled_rms_norm(float* x, const void* y1, int y1_bf16, long y1_stride, const void* y2,
                                      int y2_bf16, long y2_stride, float mult, const float* next_w, void* out,
                                      int out_bf16, int rows, int width, float eps, hipStream_t s) {
  if (rows <= 0) return 0;
  if (y1 == nullptr && (y2 != nullptr || out == nullptr)) return -1;
  if (out_bf16)
    hipLaunchKernelGGL((add_scaled_rms_norm_kernel<bf16_t, 256>), dim3(rows), dim3(256), 0, s, x, y1, y1_bf16,
                       y1_stride, y2, y2_bf16, y2_stride, mult, next_w, (bf16_t*)out, width, eps);
  else
    hipLaunchKernelGGL((add_scaled_rms_norm_kernel<float, 256>), dim3(rows), dim3(256), 0, s, x, y1, y1_bf16,
                       y1_stride, y2, y2_bf16, y2_stride, mult, next_w, (float*)out, width, eps);
  return (int)hipGetLastError();
}

extern "C" int mx_dual_rms_mean(float* out, const void* a, long a_stride, const void* b, long b_stride, int bf16,
                                const float* wa, const float* wb, int rows, int width, float eps, float scale,
                                hipStream_t s) {
  if (rows <= 0) return 0;
  MX_DISPATCH_T(bf16, hipLaunchKernelGGL((dual_rms_mean_kernel<T, 256>), dim3(rows), dim3(256), 0, s, out,
                                         (const T*)a, a_stride, (const T*)b, b_stride, wa, wb, width, eps, scale));
  return (int)hipGetLastError();
}

extern "C" int mx_sigmoid_gate(void* out, int out_bf16, const float* o, const void* g, int g_bf16, long g_stride,
                               long rows, int n, hipStream_t s) {
  if (rows * n <= 0) return 0;
  const dim3 grid(ew_grid(rows * n)), block(256);
  if (g_bf16 && out_bf16)
    hipLaunchKernelGGL((sigmoid_gate_kernel<bf16_t, bf16_t>), grid, block, 0, s, (bf16_t*)out, o, (const bf16_t*)g,
                       g_stride, rows, n);
  else if (!g_bf16 && !out_bf16)
    hipLaunchKernelGGL((sigmoid_gate_kernel<float, float>), grid, block, 0, s, (float*)out, o, (const float*)g,
                       g_stride, rows, n);
  else
    return -1;
  return (int)hipGetLastError();
}

template <typename TY, typename TO>
static void launch_shift(float* x_out, const float* x_in, const void* y, long ys, const float* wb, const float* w,
                         const float* shift, void* out, float* state, int num_slots, const int* start,
                         const int* pos0, const int* slot, int num_segs, int max_rows, int rows, int width, float eps,
                         hipStream_t s) {
  const int vec = width % 4 == 0 && (y == nullptr || (ys % 4 == 0 && ((uintptr_t)y) % (4 * sizeof(TY)) == 0)) &&
                  ((uintptr_t)x_in | (uintptr_t)x_out | (uintptr_t)w | (uintptr_t)wb | (uintptr_t)shift |
                   (uintptr_t)state) % 16 == 0 && ((uintptr_t)out) % (4 * sizeof(TO)) == 0;
  row_chunks(width, [&](auto c) {
    constexpr int C = decltype(c)::value;
    hipLaunchKernelGGL((add_norm_shift_kernel<TY, TO, kRowThreads, C>), dim3(rows), dim3(kRowThreads), 0, s, x_out,
                       x_in, (const TY*)y, ys, wb, w, shift, (TO*)out, state, num_slots, start, pos0, slot, num_segs,
                       width, eps, vec);
    if (max_rows > 1)
      hipLaunchKernelGGL((shift_state_kernel<kRowThreads, C>), dim3(num_segs), dim3(kRowThreads), 0, s, state,
                         num_slots, x_out, w, start, slot, width, eps, vec);
  });
}

extern "C" int mx_row_max_width() { return kRowMaxWidth; }

extern "C" int mx_add_norm_shift(float* x_out, const float* x_in, const void* y, int y_bf16, long y_stride,
                                 const float* wb, const float* w, const float* shift, void* out, int out_bf16,
                                 float* state, int num_slots, const int* start, const int* pos0, const int* slot,
                                 int num_segs, int max_rows, int rows, int width, float eps, hipStream_t s) {
  if (rows <= 0 || num_segs <= 0) return 0;
  if (width < 1 || width > kRowMaxWidth || (y != nullptr && max_rows > 1 && x_out == x_in)) return -1;
#define MX_SHIFT(TY, TO)                                                                                       \
  launch_shift<TY, TO>(x_out, x_in, y, y_stride, wb, w, shift, out, state, num_slots, start, pos0, slot,       \
                       num_segs, max_rows, rows, width, eps, s)
  if (y_bf16 && out_bf16) MX_SHIFT(bf16_t, bf16_t);
  else if (y_bf16) MX_SHIFT(bf16_t, float);
  else if (out_bf16) MX_SHIFT(float, bf16_t);
  else MX_SHIFT(float, float);
#undef MX_SHIFT
  return (int)hipGetLastError();
}
