// Kernels around the sequence mixers of hybrid decoders (layers that mix tokens by attention, by a recurrence, or by
// both side by side) for gfx950: embedding into a 32-bit residual stream, gated and normalised residual update, query /
// key norm + partial rotation + paged K/V write, latent norm + paged write, and row-at-a-time forms of attention and of
// per-head matrices that take any sizes.
//
// T is the type of activations and caches (bf16 raw bits or float); the residual stream, norms, gates, angles, scores
// and softmax are always fp32.  Row strides are in elements.

#include "elem.h"

namespace {
using namespace elem;

// ---- embedding: residual stream (fp32) and the first projection's input (T), both with `ld` elements per row, zero
// behind the true width.  feed[i] = r + 1 takes the token from prev_ids[r] (sampled by the previous step).  Rows are multiplied
// by `scale`; with `turns`, sine (even columns) and cosine (odd ones) of position * frequency are added.  turns[c / 2] is the
// frequency in turns as the sum of two floats, so that whole turns come off before anything is rounded.  `keep`: a second copy.
__device__ inline float2 sine_pair(int pos, float2 f) {
  const float p = (float)pos;
  const float r = fmaf(p, f.x, -rintf(p * f.x)) + p * f.y;  // (exact product less whole turns, rounded once)
  float s, c;
  sincospif(2.f * r, &s, &c);
  return make_float2(s, c);
}

template <typename T>
__global__ __launch_bounds__(256) void embed_stream_kernel(const T* __restrict__ table, const int* __restrict__ tokens, const int* __restrict__ feed,
                                                           const long long* __restrict__ prev_ids, int n_prev, float* __restrict__ x, T* __restrict__ xb, float* __restrict__ keep, float scale,
                                                           const int* __restrict__ positions, const float2* __restrict__ turns, int H, int ld, int V) {
  const int i = blockIdx.x;
  const int f = feed[i];
  long long tok = (f > 0 && f <= n_prev) ? prev_ids[f - 1] : (long long)tokens[i];
  if (tok < 0 || tok >= V) tok = 0;
  const T* src = table + tok * H;
  for (int c = threadIdx.x * 4; c < ld; c += 1024) {  // (ld is a multiple of four)
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    if ((H & 3) == 0) {
      if (c < H) v = ld4(src + c);
    } else {
      if (c < H) v.x = elem::ld(src + c);
      if (c + 1 < H) v.y = elem::ld(src + c + 1);
      if (c + 2 < H) v.z = elem::ld(src + c + 2);
      if (c + 3 < H) v.w = elem::ld(src + c + 3);
    }
    v.x *= scale; v.y *= scale; v.z *= scale; v.w *= scale;
    if (turns && c < H) {
      const float2 a = sine_pair(positions[i], turns[c >> 1]);
      v.x += a.x;
      if (c + 1 < H) v.y += a.y;
      if (c + 2 < H) {
        const float2 b = sine_pair(positions[i], turns[(c >> 1) + 1]);
        v.z += b.x;
        if (c + 3 < H) v.w += b.y;
      }
    }
    st4(x + (long long)i * ld + c, v);
    if (keep) st4(keep + (long long)i * ld + c, v);
    st4(xb + (long long)i * ld + c, v);
  }
}

// ---- one sublayer's end: x += mult * g * unit((y + bias) * sigmoid(gate + gate_bias)), unit(r) = r / sqrt(mean r^2 + eps).
// y and gate: fp32 split-K slabs (n_slabs > 0, summed here) or rows of T; y also as weighted rows (w: row t is the sum of
// w[t n + k] times row t n + k over k < n = n_slabs; rows of weight zero are not read) or nothing (p = null: x stays).
// Then the stream takes a row of join_rows and join_vec, where given, and xb receives the new stream in T — or, with
// next_g, next_g * unit(x), the next product's input.  Gains g and next_g: one number, or one per column (g_step 1).
struct RowSource { const void* p; long long ld, slab_stride; int n_slabs; const float* w; };
struct ResidualArgs {
  const float* bias; const float* gate_bias;
  const float* g; int g_step;
  const float* next_g; int next_step;
  const float* join_rows; const float* join_vec;
  float mult, eps;
  int H, ld;
};

template <typename T>
__device__ inline float4 row4(const RowSource& s, long long t, int c) {
  if (s.w) {
    float4 a = make_float4(0.f, 0.f, 0.f, 0.f);
    for (int k = 0; k < s.n_slabs; ++k) {
      const float w = s.w[t * s.n_slabs + k];
      if (w == 0.f) continue;
      const float4 b = ld4(reinterpret_cast<const T*>(s.p) + (t * s.n_slabs + k) * s.ld + c);
      a.x += w * b.x; a.y += w * b.y; a.z += w * b.z; a.w += w * b.w;
    }
    return a;
  }
  if (s.n_slabs == 0) return ld4(reinterpret_cast<const T*>(s.p) + t * s.ld + c);
  const float* p = reinterpret_cast<const float*>(s.p) + t * s.ld + c;
  float4 a = ld4(p);
#pragma unroll 4
  for (int k = 1; k < s.n_slabs; ++k) {
    const float4 b = ld4(p + (long long)k * s.slab_stride);
    a.x += b.x; a.y += b.y; a.z += b.z; a.w += b.w;
  }
  return a;
}

template <int NT>
__device__ inline float block_sum(float v, float* red) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int w = 0; w < NT / 64; ++w) s += red[w];
  return s;
}

__device__ inline float4 gain4(const float* g, int step, int c) {
  if (step) return ld4(g + c);
  return make_float4(g[0], g[0], g[0], g[0]);
}

template <typename T, int NT>
__global__ __launch_bounds__(NT) void gated_residual_kernel(float* __restrict__ x, T* __restrict__ xb, RowSource y, RowSource gate, ResidualArgs a) {
  extern __shared__ __attribute__((aligned(16))) float row[];  // ld floats
  __shared__ float red[NT / 64];
  const long long t = blockIdx.x;
  const int ld = a.ld;
  const float inv_h = 1.f / (float)a.H;
  float k = 0.f;
  // (columns H .. ld: weights, biases and stream are zero there, so every term is)
  if (y.p) {
    float ss = 0.f;
    for (int c = threadIdx.x * 4; c < ld; c += NT * 4) {
      float4 v = row4<T>(y, t, c);
      if (a.bias) { const float4 b = ld4(a.bias + c); v.x += b.x; v.y += b.y; v.z += b.z; v.w += b.w; }
      if (gate.p) {
        float4 z = row4<T>(gate, t, c);
        const float4 b = ld4(a.gate_bias + c);
        v.x *= sigmoid(z.x + b.x); v.y *= sigmoid(z.y + b.y); v.z *= sigmoid(z.z + b.z); v.w *= sigmoid(z.w + b.w);
      }
      ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
      st4(row + c, v);
    }
    k = a.mult / sqrtf(block_sum<NT>(ss, red) * inv_h + a.eps);
  }
  float* xr = x + t * ld;
  float xs = 0.f;
  for (int c = threadIdx.x * 4; c < ld; c += NT * 4) {
    float4 v = ld4(xr + c);
    if (y.p) {
      const float4 r = ld4(row + c), g = gain4(a.g, a.g_step, c);
      v.x += k * g.x * r.x; v.y += k * g.y * r.y; v.z += k * g.z * r.z; v.w += k * g.w * r.w;
    }
    if (a.join_vec) {
      float4 j = ld4(a.join_vec + c);
      if (a.join_rows) { const float4 e = ld4(a.join_rows + t * ld + c); j.x += e.x; j.y += e.y; j.z += e.z; j.w += e.w; }
      v.x += j.x; v.y += j.y; v.z += j.z; v.w += j.w;
    }
    st4(xr + c, v);
    if (a.next_g) {
      xs += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
      st4(row + c, v);
    } else {
      st4(xb + t * ld + c, v);
    }
  }
  if (!a.next_g) return;
  const float f = 1.f / sqrtf(block_sum<NT>(xs, red) * inv_h + a.eps);
  for (int c = threadIdx.x * 4; c < ld; c += NT * 4) {
    float4 v = ld4(row + c);
    const float4 g = gain4(a.next_g, a.next_step, c);
    v.x *= f * g.x; v.y *= f * g.y; v.z *= f * g.z; v.w *= f * g.w;
    st4(xb + t * ld + c, v);
  }
}

// ---- the end of a layer whose mixer and feed-forward read the same stream: x += y + bias + y2 + y3 (rows as above, whichever are given);
// xb and xb2 receive g * unit(x) and g2 * unit(x), the next layer's inputs (no g2: xb alone).
struct ParallelArgs { const float* bias; const float* g; const float* g2; float eps; int H, ld; };

template <typename T, int NT>
__global__ __launch_bounds__(NT) void parallel_residual_kernel(float* __restrict__ x, T* __restrict__ xb, T* __restrict__ xb2, RowSource y, RowSource y2, RowSource y3, ParallelArgs a) {
  extern __shared__ __attribute__((aligned(16))) float row[];  // ld floats
  __shared__ float red[NT / 64];
  const long long t = blockIdx.x;
  const int ld = a.ld;
  float* xr = x + t * ld;
  const bool more = y.p || y2.p || y3.p || a.bias;
  float ss = 0.f;
  auto add = [](float4& v, float4 b) __attribute__((always_inline)) { v.x += b.x; v.y += b.y; v.z += b.z; v.w += b.w; };
  for (int c = threadIdx.x * 4; c < ld; c += NT * 4) {
    float4 v = ld4(xr + c);
    if (more) {
      float4 r = make_float4(0.f, 0.f, 0.f, 0.f);
      if (y.p) add(r, row4<T>(y, t, c));
      if (y3.p) add(r, row4<T>(y3, t, c));
      if (y2.p) add(r, row4<T>(y2, t, c));
      if (a.bias) add(r, ld4(a.bias + c));
      add(v, r);
      st4(xr + c, v);
    }
    ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;  // (columns H .. ld are zero)
    st4(row + c, v);
  }
  const float f = 1.f / sqrtf(block_sum<NT>(ss, red) / (float)a.H + a.eps);
  for (int c = threadIdx.x * 4; c < ld; c += NT * 4) {
    float4 v = ld4(row + c);
    v.x *= f; v.y *= f; v.z *= f; v.w *= f;
    const float4 g = ld4(a.g + c);
    st4(xb + t * ld + c, make_float4(v.x * g.x, v.y * g.y, v.z * g.z, v.w * g.w));
    if (a.g2) {
      const float4 k = ld4(a.g2 + c);
      st4(xb2 + t * ld + c, make_float4(v.x * k.x, v.y * k.y, v.z * k.z, v.w * k.w));
    }
  }
}

// ---- the end of a sublayer between several streams: every stream becomes sum_s mix[s][t] x_s + out[t] y (y: rows as above, plus gate2[row]
// times the rows y2), or, without y, a copy of `start` or what it is; xb receives next_g * unit(sum_t read[t] x_t).  NS: streams at most
// (EXACT: just as many).
struct HyperArgs {
  int n;
  const float* mix; const float* out; const float* read;
  const float* next_g; const float* start; const float* gate2;
  float eps;
  int H, ld;
};

template <typename T, int NT, int NS, bool EXACT>
__global__ __launch_bounds__(NT) void hyper_residual_kernel(float* __restrict__ x, T* __restrict__ xb, RowSource y, RowSource y2, HyperArgs a) {
  extern __shared__ __attribute__((aligned(16))) float row[];  // ld floats
  __shared__ float red[NT / 64];
  const long long t = blockIdx.x;
  const int ld = a.ld, n = EXACT ? NS : a.n;
  float* xr = x + t * n * ld;
  const float f2 = y2.p ? a.gate2[t] : 0.f;
  float ss = 0.f;
  for (int c = threadIdx.x * 4; c < ld; c += NT * 4) {
    float4 s[NS];
#pragma unroll
    for (int i = 0; i < NS; ++i)
      if (i < n) s[i] = a.start ? ld4(a.start + t * ld + c) : ld4(xr + (long long)i * ld + c);
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f), u = v;
    if (y.p) v = row4<T>(y, t, c);
    if (y2.p) {
      const float4 w = row4<T>(y2, t, c);
      v.x += f2 * w.x; v.y += f2 * w.y; v.z += f2 * w.z; v.w += f2 * w.w;
    }
#pragma unroll
    for (int j = 0; j < NS; ++j) {
      if (j >= n) break;
      float4 z = s[j];
      if (y.p) {
        const float o = a.out[j];
        z = make_float4(o * v.x, o * v.y, o * v.z, o * v.w);
#pragma unroll
        for (int i = 0; i < NS; ++i)
          if (i < n) {
            const float m = a.mix[i * n + j];
            z.x += m * s[i].x; z.y += m * s[i].y; z.z += m * s[i].z; z.w += m * s[i].w;
          }
      }
      if (y.p || a.start) st4(xr + (long long)j * ld + c, z);
      const float r = a.read[j];
      u.x += r * z.x; u.y += r * z.y; u.z += r * z.z; u.w += r * z.w;
    }
    ss += u.x * u.x + u.y * u.y + u.z * u.z + u.w * u.w;  // (columns H .. ld are zero)
    st4(row + c, u);
  }
  const float f = 1.f / sqrtf(block_sum<NT>(ss, red) / (float)a.H + a.eps);
  for (int c = threadIdx.x * 4; c < ld; c += NT * 4) {
    float4 u = ld4(row + c);
    const float4 g = ld4(a.next_g + c);
    st4(xb + t * ld + c, make_float4(u.x * f * g.x, u.y * f * g.y, u.z * f * g.z, u.w * f * g.w));
  }
}

// ---- cap * tanh(logit / cap), in place
template <typename T>
__global__ __launch_bounds__(256) void softcap_kernel(T* __restrict__ x, long long stride, int V, float cap, float inv_cap) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= V) return;
  T* p = x + blockIdx.y * stride + c;
  st(p, cap * tanhf(ld(p) * inv_cap));
}

// ---- query / key norm, rotation of the first rot_dims dimensions, paged K/V write.  One wave per (token, head); heads in
// the order query heads, key heads, value heads.  q [T, nh, dkp], caches [blocks, nkv, block_size, dkp | dvp]; dimensions
// behind dim / vdim are written as zero.
struct NormRopeArgs {
  long long ldp; int q_off, k_off, v_off;
  const float* bias;  // [nh dim + nkv dim + nkv vdim] or null
  const float* q_norm; const float* k_norm;  // [dim] or null
  const int* positions; const int* slots;
  const float* cos_t; const float* sin_t;  // [max_pos, rot_dims / 2]
  int rot_dims, nh, nkv, dim, vdim, dkp, dvp, block_size;
  float eps;
};

template <typename T>
__global__ __launch_bounds__(256) void norm_rope_write_kernel(const T* __restrict__ proj, T* __restrict__ q, T* __restrict__ k_cache, T* __restrict__ v_cache, NormRopeArgs a) {
  extern __shared__ float buf[];  // 4 x dim
  const long long t = blockIdx.x;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int unit = blockIdx.y * 4 + wave, n_units = a.nh + 2 * a.nkv;
  const bool on = unit < n_units;
  const bool is_q = unit < a.nh, is_v = unit >= a.nh + a.nkv;
  const int head = is_q ? unit : is_v ? unit - a.nh - a.nkv : unit - a.nh;
  const int n = is_v ? a.vdim : a.dim;
  const T* src = proj + t * a.ldp + (is_q ? a.q_off : is_v ? a.v_off : a.k_off) + head * n;
  const int b_off = is_q ? head * n : is_v ? (a.nh + a.nkv) * a.dim + head * n : (a.nh + head) * n;
  const int slot = a.slots[t];
  const int pos = a.positions[t];
  float* w = buf + wave * a.dim;
  const int half = a.rot_dims >> 1;
  if (on && !is_v) {
    float ss = 0.f;
    for (int i = lane; i < n; i += 64) {
      const float v = ld(src + i) + (a.bias ? a.bias[b_off + i] : 0.f);
      w[i] = v;
      ss += v * v;
    }
    const float* nw = is_q ? a.q_norm : a.k_norm;
    if (nw) {
      const float rs = 1.f / sqrtf(wave_sum(ss) / (float)n + a.eps);
      for (int i = lane; i < n; i += 64) w[i] = w[i] * rs * nw[i];
    }
  }
  __syncthreads();
  if (!on) return;
  if (!is_q && slot < 0) return;
  const int np = is_v ? a.dvp : a.dkp;
  T* dst;
  if (is_q) dst = q + (t * a.nh + head) * np;
  else dst = (is_v ? v_cache : k_cache) + (((long long)(slot / a.block_size) * a.nkv + head) * a.block_size + slot % a.block_size) * np;
  for (int i = lane; i < np; i += 64) {
    float v = 0.f;
    if (i < n) {
      if (is_v) {
        v = ld(src + i) + (a.bias ? a.bias[b_off + i] : 0.f);
      } else if (i < a.rot_dims) {
        const int p = i < half ? i : i - half;
        const float c = a.cos_t[(long long)pos * half + p], s = a.sin_t[(long long)pos * half + p];
        v = i < half ? w[i] * c - w[i + half] * s : w[i] * c + w[i - half] * s;
      } else {
        v = w[i];
      }
    }
    st(dst + i, v);
  }
}

// The same for head sizes in eights (bf16; sections, rotated half and padded sizes multiples of 8): LPR lanes per head, 8 elements
// (16 bytes) each, the partner of a rotated element sits rot_dims / 16 lanes away at the same index.
template <int LPR>
__global__ __launch_bounds__(256) void norm_rope_write_vec_kernel(const bf16raw* __restrict__ proj, bf16raw* __restrict__ q, bf16raw* __restrict__ k_cache, bf16raw* __restrict__ v_cache,
                                                                  NormRopeArgs a) {
  typedef __attribute__((ext_vector_type(8))) unsigned short us8;
  const long long t = blockIdx.x;
  const int unit = blockIdx.y * (256 / LPR) + threadIdx.x / LPR, lane = threadIdx.x % LPR, n_units = a.nh + 2 * a.nkv;
  if (unit >= n_units) return;  // (whole groups of LPR lanes: the exchanges below stay inside a group)
  const bool is_q = unit < a.nh, is_v = unit >= a.nh + a.nkv;
  const int head = is_q ? unit : is_v ? unit - a.nh - a.nkv : unit - a.nh;
  const int n = is_v ? a.vdim : a.dim, np = is_v ? a.dvp : a.dkp;
  const int slot = a.slots[t], pos = a.positions[t];
  const int i0 = lane * 8;
  const bool on = i0 < n;
  float x[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) x[e] = 0.f;
  if (on) {
    const us8 v = *reinterpret_cast<const us8*>(proj + t * a.ldp + (is_q ? a.q_off : is_v ? a.v_off : a.k_off) + head * n + i0);
    const float* b = a.bias ? a.bias + (is_q ? head * n : is_v ? (a.nh + a.nkv) * a.dim + head * n : (a.nh + head) * n) + i0 : nullptr;
    float bv[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (b) { *reinterpret_cast<float4*>(bv) = ld4(b); *reinterpret_cast<float4*>(bv + 4) = ld4(b + 4); }
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] = bf2f(v[e]) + bv[e];
  }
  if (!is_v) {
    const float* nw = is_q ? a.q_norm : a.k_norm;
    if (nw) {
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += x[e] * x[e];
#pragma unroll
      for (int m = 1; m < LPR; m <<= 1) ss += __shfl_xor(ss, m, 64);
      const float rs = 1.f / sqrtf(ss / (float)n + a.eps);
      if (on) {
        float nv[8];
        *reinterpret_cast<float4*>(nv) = ld4(nw + i0);
        *reinterpret_cast<float4*>(nv + 4) = ld4(nw + i0 + 4);
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] *= rs * nv[e];
      }
    }
    const int half = a.rot_dims >> 1, hl = half >> 3;
    if (half > 0) {
      const bool low = i0 < half, rot = i0 < a.rot_dims;
      const int partner = (threadIdx.x & 63) + (rot ? (low ? hl : -hl) : 0);
      const int p0 = rot ? (low ? i0 : i0 - half) : 0;
      float cv[8], sv[8];
#pragma unroll
      for (int e = 0; e < 8; e += 4) {
        *reinterpret_cast<float4*>(cv + e) = ld4(a.cos_t + (long long)pos * half + p0 + e);
        *reinterpret_cast<float4*>(sv + e) = ld4(a.sin_t + (long long)pos * half + p0 + e);
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float y = __shfl(x[e], partner, 64);
        if (rot) x[e] = low ? x[e] * cv[e] - y * sv[e] : x[e] * cv[e] + y * sv[e];
      }
    }
  }
  if ((!is_q && slot < 0) || i0 >= np) return;
  bf16raw* dst;
  if (is_q) dst = q + (t * a.nh + head) * np;
  else dst = (is_v ? v_cache : k_cache) + (((long long)(slot / a.block_size) * a.nkv + head) * a.block_size + slot % a.block_size) * np;
  us8 o;
#pragma unroll
  for (int e = 0; e < 8; ++e) o[e] = f2bf(x[e]);
  *reinterpret_cast<us8*>(dst + i0) = o;
}

// ---- the same where the values are the keys as projected (bf16): a cache row is [key as it is, dvp | its first rot_dims dimensions, rotated, rt],
// key_scale[row] the factor that norms the key.  Query rows are [0 in the first rot_dims, the others normed and times the keys' gains, dvp | the
// first ones normed and rotated, rt].  Heads in the order query heads, key heads; v_off, vdim, dkp, v_cache of the arguments are not used.
template <int LPR>  // lanes per head, 8 elements each (sizes as for norm_rope_write_vec_kernel)
__global__ __launch_bounds__(256) void key_value_write_vec_kernel(const bf16raw* __restrict__ proj, bf16raw* __restrict__ q, bf16raw* __restrict__ cache, float* __restrict__ key_scale, int rt, NormRopeArgs a) {
  typedef __attribute__((ext_vector_type(8))) unsigned short us8;
  const long long t = blockIdx.x;
  const int unit = blockIdx.y * (256 / LPR) + threadIdx.x / LPR, lane = threadIdx.x % LPR;
  if (unit >= a.nh + a.nkv) return;  // (whole groups of LPR lanes: the exchanges below stay inside a group)
  const bool is_q = unit < a.nh;
  const int head = is_q ? unit : unit - a.nh;
  const int slot = a.slots[t], pos = a.positions[t];
  const int i0 = lane * 8;
  const bool on = i0 < a.dim;
  float x[8], kg[8], qg[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) x[e] = kg[e] = qg[e] = 0.f;
  if (on) {
    const us8 v = *reinterpret_cast<const us8*>(proj + t * a.ldp + (is_q ? a.q_off : a.k_off) + head * a.dim + i0);
    const float* b = a.bias + (is_q ? head : a.nh + head) * a.dim + i0;
    float bv[8];
    *reinterpret_cast<float4*>(bv) = ld4(b);
    *reinterpret_cast<float4*>(bv + 4) = ld4(b + 4);
    *reinterpret_cast<float4*>(kg) = ld4(a.k_norm + i0);
    *reinterpret_cast<float4*>(kg + 4) = ld4(a.k_norm + i0 + 4);
    *reinterpret_cast<float4*>(qg) = ld4(a.q_norm + i0);
    *reinterpret_cast<float4*>(qg + 4) = ld4(a.q_norm + i0 + 4);
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] = bf2f(v[e]) + bv[e];
  }
  float ss = 0.f;
#pragma unroll
  for (int e = 0; e < 8; ++e) ss += x[e] * x[e];
#pragma unroll
  for (int m = 1; m < LPR; m <<= 1) ss += __shfl_xor(ss, m, 64);
  const float rs = 1.f / sqrtf(ss / (float)a.dim + a.eps);
  float w[8];  // what turns: the normed query, or the key with its gains
#pragma unroll
  for (int e = 0; e < 8; ++e) w[e] = x[e] * (is_q ? rs * qg[e] : kg[e]);
  const bool rot = i0 < a.rot_dims;
  us8 straight, turned;
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    straight[e] = is_q ? (rot ? (bf16raw)0 : f2bf(w[e] * kg[e])) : f2bf(x[e]);
    turned[e] = 0;
  }
  const int half = a.rot_dims >> 1, hl = half >> 3;
  if (half > 0) {
    const bool low = i0 < half;
    const int partner = (threadIdx.x & 63) + (rot ? (low ? hl : -hl) : 0);
    const int p0 = rot ? (low ? i0 : i0 - half) : 0;
    float cv[8], sv[8];
#pragma unroll
    for (int e = 0; e < 8; e += 4) {
      *reinterpret_cast<float4*>(cv + e) = ld4(a.cos_t + (long long)pos * half + p0 + e);
      *reinterpret_cast<float4*>(sv + e) = ld4(a.sin_t + (long long)pos * half + p0 + e);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float y = __shfl(w[e], partner, 64);
      if (rot) turned[e] = f2bf(low ? w[e] * cv[e] - y * sv[e] : w[e] * cv[e] + y * sv[e]);
    }
  }
  if (!is_q && slot < 0) return;
  const int np = a.dvp + rt;
  const long long row = is_q ? t * a.nh + head : ((long long)(slot / a.block_size) * a.nkv + head) * a.block_size + slot % a.block_size;
  bf16raw* dst = (is_q ? q : cache) + row * np;
  if (i0 < a.dvp) *reinterpret_cast<us8*>(dst + i0) = straight;
  if (i0 < rt) *reinterpret_cast<us8*>(dst + a.dvp + i0) = turned;
  if (!is_q && lane == 0) key_scale[row] = rs;
}

__global__ __launch_bounds__(256) void key_value_write_kernel(const bf16raw* __restrict__ proj, bf16raw* __restrict__ q, bf16raw* __restrict__ cache, float* __restrict__ key_scale, int rt, NormRopeArgs a) {
  extern __shared__ float buf[];  // 4 x dim
  const long long t = blockIdx.x;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int unit = blockIdx.y * 4 + wave;
  const bool on = unit < a.nh + a.nkv, is_q = unit < a.nh;
  const int head = is_q ? unit : unit - a.nh;
  const bf16raw* src = proj + t * a.ldp + (is_q ? a.q_off : a.k_off) + head * a.dim;
  const float* bias = a.bias + (is_q ? head : a.nh + head) * a.dim;
  const int slot = a.slots[t], pos = a.positions[t], half = a.rot_dims >> 1;
  float* w = buf + wave * a.dim;
  float rs = 1.f;
  if (on) {
    float ss = 0.f;
    for (int i = lane; i < a.dim; i += 64) {
      const float v = ld(src + i) + bias[i];
      w[i] = v;
      ss += v * v;
    }
    rs = 1.f / sqrtf(wave_sum(ss) / (float)a.dim + a.eps);
    for (int i = lane; i < a.dim; i += 64) w[i] *= is_q ? rs * a.q_norm[i] : a.k_norm[i];
  }
  __syncthreads();
  if (!on || (!is_q && slot < 0)) return;
  const long long row = is_q ? t * a.nh + head : ((long long)(slot / a.block_size) * a.nkv + head) * a.block_size + slot % a.block_size;
  bf16raw* dst = (is_q ? q : cache) + row * (a.dvp + rt);
  for (int i = lane; i < a.dvp; i += 64) st(dst + i, i >= a.dim ? 0.f : !is_q ? ld(src + i) + bias[i] : i < a.rot_dims ? 0.f : w[i] * a.k_norm[i]);
  for (int i = lane; i < rt; i += 64) {
    float v = 0.f;
    if (i < a.rot_dims) {
      const int p = i < half ? i : i - half;
      const float c = a.cos_t[(long long)pos * half + p], s = a.sin_t[(long long)pos * half + p];
      v = i < half ? w[i] * c - w[i + half] * s : w[i] * c + w[i - half] * s;
    }
    st(dst + a.dvp + i, v);
  }
  if (!is_q && lane == 0) key_scale[row] = rs;
}

// ---- latent attention's cache entry: gain * unit(latent), one wave per row; columns behind `rank` have gain zero.  With a rotated part
// (rot), the key part follows it in the cache, and the workgroups with blockIdx.y = 1 rotate the rows' query parts (into dst, which may be
// where they are).  Neighbouring elements 2i, 2i + 1 turn together; columns rot .. rtp become zero.
struct LatentWriteArgs {
  long long ldp; int c_off;
  const float* gain; const int* slots; const int* positions;
  int n_rows, rank, rkp, write;
  int rot, rtp, kr_off; const float* cos_t; const float* sin_t;  // [positions][rot / 2]
  int nh, r_off; long long ldd; int d_off, d_head;
  float eps;
};

__device__ inline float2 turn(float2 v, float c, float s) { return make_float2(v.x * c - v.y * s, v.y * c + v.x * s); }

template <typename T>
__global__ __launch_bounds__(256) void latent_write_kernel(const T* proj, T* __restrict__ cache, T* dst, LatentWriteArgs a) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (t >= a.n_rows) return;
  const int slot = a.slots[t];
  if (slot < 0) return;
  const T* row = proj + (long long)t * a.ldp;
  const int half = a.rot >> 1, halfp = a.rtp >> 1;
  const float* ct = a.cos_t + (long long)(half ? a.positions[t] : 0) * half;
  const float* st_ = a.sin_t + (long long)(half ? a.positions[t] : 0) * half;
  if (blockIdx.y == 1) {
    for (int i = lane; i < a.nh * halfp; i += 64) {
      const int h = i / halfp, p = i - h * halfp;
      const T* q = row + a.r_off + h * a.rtp + 2 * p;
      float2 v = make_float2(0.f, 0.f);
      if (p < half) v = turn(make_float2(ld(q), ld(q + 1)), ct[p], st_[p]);
      T* o = dst + (long long)t * a.ldd + a.d_off + h * a.d_head + 2 * p;
      st(o, v.x);
      st(o + 1, v.y);
    }
    return;
  }
  if (!a.write) return;
  const T* src = row + a.c_off;
  T* out = cache + (long long)slot * (a.rkp + a.rtp);
  float4 v[4];  // (rkp <= 1024)
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = (lane + 64 * i) * 4;
    v[i] = c < a.rkp ? ld4(src + c) : make_float4(0.f, 0.f, 0.f, 0.f);
    ss += v[i].x * v[i].x + v[i].y * v[i].y + v[i].z * v[i].z + v[i].w * v[i].w;
  }
  const float rs = 1.f / sqrtf(wave_sum(ss) / (float)a.rank + a.eps);
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = (lane + 64 * i) * 4;
    if (c >= a.rkp) continue;
    const float4 g = ld4(a.gain + c);
    st4(out + c, make_float4(v[i].x * rs * g.x, v[i].y * rs * g.y, v[i].z * rs * g.z, v[i].w * rs * g.w));
  }
  for (int p = lane; p < halfp; p += 64) {
    float2 k = make_float2(0.f, 0.f);
    if (p < half) k = turn(make_float2(ld(row + a.kr_off + 2 * p), ld(row + a.kr_off + 2 * p + 1)), ct[p], st_[p]);
    st(out + a.rkp + 2 * p, k.x);
    st(out + a.rkp + 2 * p + 1, k.y);
  }
}

// ---- one matrix per head, row by row: out[t][h][n] = f sum_k w[h][n][k] x[t][h][k] for n < n_true, f = out_scale times, with a
// gate, sigmoid(gate[t][h]) (gated 1) or sigmoid(gate[t][h n_true + n]) (2).  Serves every size, fp32 as well as bf16; one workgroup per (row, head).
struct HeadRowsArgs {
  long long ldx; int x_off, x_head;  // row stride, first column, columns per head
  long long ldo; int o_off, o_head;
  long long ld_gate; int gate_off, gated;
  int N, K, n_true;
  float out_scale;
  const int* slots;
};

template <typename T>
__global__ __launch_bounds__(256) void head_rows_kernel(const T* __restrict__ x, const T* __restrict__ w, const T* __restrict__ gate, T* __restrict__ out, HeadRowsArgs a) {
  extern __shared__ float sm[];  // K floats
  const long long t = blockIdx.x;
  const int h = blockIdx.y, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  T* o = out + t * a.ldo + a.o_off + (long long)h * a.o_head;
  if (a.slots[t] < 0) {  // padding row
    for (int n = threadIdx.x; n < a.n_true; n += 256) st(o + n, 0.f);
    return;
  }
  for (int k = threadIdx.x; k < a.K; k += 256) sm[k] = ld(x + t * a.ldx + a.x_off + (long long)h * a.x_head + k);
  __syncthreads();
  float f = a.out_scale;
  if (a.gated == 1) f *= sigmoid(ld(gate + t * a.ld_gate + a.gate_off + h));
  for (int n = wave; n < a.n_true; n += 4) {
    const T* wr = w + ((long long)h * a.N + n) * a.K;
    float s = 0.f;
    for (int k = lane; k < a.K; k += 64) s += ld(wr + k) * sm[k];
    s = wave_sum(s);
    if (lane == 0) st(o + n, s * (a.gated == 2 ? f * sigmoid(ld(gate + t * a.ld_gate + a.gate_off + (long long)h * a.n_true + n)) : f));
  }
}

// ---- attention of single rows: one wave per (listed row, query head), keys in blocks of 64.  A row at position p sees
// keys [p - p % chunk, p] (chunk = 0: [0, p]) or, with a window, the last `window` ones up to p and the first `keep` ones.  rel: rel[head][distance]
// (the last entry: and beyond) is added to the scaled scores; sink: the denominator has one more term exp(sink[head]).  The head's output is
// multiplied by out_scale and, with a gate, by sigmoid(gate[row][head]) (gated 1) or sigmoid(gate[row][head vdim + i]) (2).  Serves every head size up to 1024, fp32 as well as bf16.
struct RowAttentionArgs {
  const int* block_tables; int max_blocks;
  const int* tok_seq; const int* positions; const int* slots;
  int nh, nkv, dkp, vdim, dvp, block_size, chunk, window, keep;
  const float* sink; const float* rel; int rel_n;
  float scale, out_scale;
  long long ld_gate; int gate_off, gated;
  long long ldo; int o_off;
  int only_flag; const int* row_flag;  // only_flag >= 0: only rows with row_flag[t] == only_flag
};

template <typename T, int NV>
__global__ __launch_bounds__(64) void row_attention_kernel(const T* __restrict__ q, const T* __restrict__ k_cache, const T* __restrict__ v_cache, const T* __restrict__ gate,
                                                           T* __restrict__ out, RowAttentionArgs a) {
  extern __shared__ float sm[];  // q: dkp floats, then 64 probabilities
  const long long t = blockIdx.x;
  const int h = blockIdx.y, lane = threadIdx.x;
  if (a.only_flag >= 0 && a.row_flag[t] != a.only_flag) return;
  T* o = out + t * a.ldo + a.o_off + h * a.vdim;
  if (a.slots[t] < 0) {  // padding row
    for (int i = lane; i < a.vdim; i += 64) st(o + i, 0.f);
    return;
  }
  float* qs = sm;
  float* ps = sm + a.dkp;
  for (int i = lane; i < a.dkp; i += 64) qs[i] = ld(q + (t * a.nh + h) * a.dkp + i);
  __syncthreads();
  const int g = h / (a.nh / a.nkv);
  const int pos = a.positions[t];
  const int first = a.window > 0 ? (pos >= a.window ? pos - a.window + 1 : 0) : a.chunk > 0 ? pos - pos % a.chunk : 0;
  const int* bt = a.block_tables + (long long)a.tok_seq[t] * a.max_blocks;
  const int kept = a.keep < first ? a.keep : first, n_keys = kept + pos - first + 1;  // keys 0 .. kept, first .. pos
  float m = a.sink ? a.sink[h] : -INFINITY, l = a.sink ? 1.f : 0.f, acc[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) acc[i] = 0.f;
  for (int kb = 0; kb < n_keys; kb += 64) {
    const int ki = kb + lane, key = ki < kept ? ki : first + ki - kept;
    float s = -INFINITY;
    if (ki < n_keys) {
      const T* kr = k_cache + (((long long)bt[key / a.block_size] * a.nkv + g) * a.block_size + key % a.block_size) * a.dkp;
      float d = 0.f;
      for (int i = 0; i < a.dkp; i += 4) {
        const float4 kv = ld4(kr + i);
        const float4 qv = ld4(qs + i);
        d += kv.x * qv.x + kv.y * qv.y + kv.z * qv.z + kv.w * qv.w;
      }
      s = d * a.scale;
      if (a.rel) s += a.rel[(long long)h * a.rel_n + (pos - key < a.rel_n ? pos - key : a.rel_n - 1)];
    }
    const float m_new = fmaxf(m, wave_max(s));
    const float p = ki < n_keys ? expf(s - m_new) : 0.f;
    const float corr = expf(m - m_new);
    l = l * corr + wave_sum(p);
    m = m_new;
    __syncthreads();
    ps[lane] = p;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NV; ++i) acc[i] *= corr;
    const int nk = n_keys - kb < 64 ? n_keys - kb : 64;
    for (int j = 0; j < nk; ++j) {
      const int kk = kb + j < kept ? kb + j : first + kb + j - kept;
      const T* vr = v_cache + (((long long)bt[kk / a.block_size] * a.nkv + g) * a.block_size + kk % a.block_size) * a.dvp;
      const float pj = ps[j];
#pragma unroll
      for (int i = 0; i < NV; ++i)
        if (lane + 64 * i < a.vdim) acc[i] += pj * ld(vr + lane + 64 * i);
    }
  }
  float f = a.out_scale / l;
  if (a.gated == 1) f *= sigmoid(ld(gate + t * a.ld_gate + a.gate_off + h));
#pragma unroll
  for (int i = 0; i < NV; ++i)
    if (lane + 64 * i < a.vdim) st(o + lane + 64 * i, acc[i] * (a.gated == 2 ? f * sigmoid(ld(gate + t * a.ld_gate + a.gate_off + h * a.vdim + lane + 64 * i)) : f));
}

// ---- index of the largest entry of every row (the first one of equals), fp32 logits
__global__ __launch_bounds__(1024) void argmax_f32_kernel(const float* __restrict__ logits, long long stride, int V, long long* __restrict__ out) {
  __shared__ float bv[16];
  __shared__ int bi[16];
  const float* row = logits + (long long)blockIdx.x * stride;
  float best = -INFINITY;
  int idx = 0x7fffffff;
  for (int i = threadIdx.x; i < V; i += 1024) {
    const float v = row[i];
    if (v > best || (v == best && i < idx)) { best = v; idx = i; }
  }
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float v = __shfl_xor(best, o, 64);
    const int i = __shfl_xor(idx, o, 64);
    if (v > best || (v == best && i < idx)) { best = v; idx = i; }
  }
  if ((threadIdx.x & 63) == 0) { bv[threadIdx.x >> 6] = best; bi[threadIdx.x >> 6] = idx; }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < 16; ++w)
      if (bv[w] > best || (bv[w] == best && bi[w] < idx)) { best = bv[w]; idx = bi[w]; }
    out[blockIdx.x] = idx < V ? idx : 0;
  }
}

template <typename T>
int launch_row_attention(const void* q, const void* kc, const void* vc, const void* gate, void* out, int T_, const RowAttentionArgs& a, hipStream_t s) {
  const size_t lds = (size_t)(a.dkp + 64) * 4;
  const dim3 grid(T_, a.nh);
#define KV_RA(NV) hipLaunchKernelGGL((row_attention_kernel<T, NV>), grid, dim3(64), lds, s, (const T*)q, (const T*)kc, (const T*)vc, (const T*)gate, (T*)out, a)
  if (a.vdim <= 64) KV_RA(1);
  else if (a.vdim <= 128) KV_RA(2);
  else if (a.vdim <= 256) KV_RA(4);
  else if (a.vdim <= 1024) KV_RA(16);
  else return -1;
#undef KV_RA
  return (int)hipGetLastError();
}

}  // namespace

extern "C" {

int kvm_embed_stream(const void* table, int f32, const int* tokens, const int* feed, const long long* prev_ids, int n_prev, float* x, void* xb, float* keep, float scale,
                     const int* positions, const float* turns, int T, int H, int ld, int V, hipStream_t s) {
  if (T <= 0 || H <= 0 || ld < H || (ld & 3) || V <= 0 || (turns && !positions)) return -1;
#define KV_ES(Tt) hipLaunchKernelGGL((embed_stream_kernel<Tt>), dim3(T), dim3(256), 0, s, (const Tt*)table, tokens, feed, prev_ids, n_prev, x, (Tt*)xb, keep, scale, positions, (const float2*)turns, H, ld, V)
  if (f32) KV_ES(float);
  else KV_ES(bf16raw);
#undef KV_ES
  return (int)hipGetLastError();
}

int kvm_gated_residual(float* x, void* xb, int f32, const void* y, long long y_ld, long long y_stride, int y_slabs, const float* y_weights, const float* bias, const void* gate,
                       long long gate_ld, long long gate_stride, int gate_slabs, const float* gate_bias, const float* g, int g_step, const float* next_g, int next_step,
                       const float* join_rows, const float* join_vec, float mult, float eps, int T, int H, int ld, hipStream_t s) {
  if (T <= 0 || H <= 0 || ld < H || (ld & 3) || ld > 32768 || (y_ld & 3) || (y && !g) || (y_weights && y_slabs < 1) || (join_rows && !join_vec) || (gate && ((gate_ld & 3) || !gate_bias))) return -1;
  const RowSource ys{y, y_ld, y_stride, y_slabs, y_weights}, gs{gate, gate_ld, gate_stride, gate_slabs, nullptr};
  const ResidualArgs a{bias, gate_bias, g, g_step, next_g, next_step, join_rows, join_vec, mult, eps, H, ld};
  const size_t lds = (size_t)ld * 4;
#define KV_GR(Tt, NT)                                                                                                                                             \
  do {                                                                                                                                                            \
    if (lds > 65536 && hipFuncSetAttribute((const void*)gated_residual_kernel<Tt, NT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) return -1; \
    hipLaunchKernelGGL((gated_residual_kernel<Tt, NT>), dim3(T), dim3(NT), lds, s, x, (Tt*)xb, ys, gs, a);                                                          \
  } while (0)
  if (ld <= 1024) { if (f32) KV_GR(float, 256); else KV_GR(bf16raw, 256); }
  else if (T <= 128) { if (f32) KV_GR(float, 1024); else KV_GR(bf16raw, 1024); }  // few rows: the whole row at once
  else { if (f32) KV_GR(float, 512); else KV_GR(bf16raw, 512); }
#undef KV_GR
  return (int)hipGetLastError();
}

int kvm_norm_rope_write(const void* proj, int f32, void* q, void* k_cache, void* v_cache, long long ldp, int q_off, int k_off, int v_off, const float* bias, const float* q_norm,
                        const float* k_norm, const int* positions, const int* slots, const float* cos_t, const float* sin_t, int rot_dims, int T, int nh, int nkv, int dim, int vdim,
                        int dkp, int dvp, int block_size, float eps, hipStream_t s) {
  if (T <= 0 || nh <= 0 || nkv <= 0 || nh % nkv || dim <= 0 || dim > 1024 || vdim <= 0 || dkp < dim || dvp < vdim || rot_dims < 0 || rot_dims > dim || (rot_dims & 1) || block_size <= 0) return -1;
  const NormRopeArgs a{ldp, q_off, k_off, v_off, bias, q_norm, k_norm, positions, slots, cos_t, sin_t, rot_dims, nh, nkv, dim, vdim, dkp, dvp, block_size, eps};
  const int widest = dkp > dvp ? dkp : dvp;
  if (!f32 && !((dim | vdim | dkp | dvp | q_off | k_off | v_off) & 7) && !(rot_dims & 15) && !(ldp & 7) && !((uintptr_t)proj & 15) && widest <= 512) {
#define KV_NR(LPR) \
  hipLaunchKernelGGL((norm_rope_write_vec_kernel<LPR>), dim3(T, (nh + 2 * nkv + 256 / LPR - 1) / (256 / LPR)), dim3(256), 0, s, (const bf16raw*)proj, (bf16raw*)q, (bf16raw*)k_cache, (bf16raw*)v_cache, a)
    if (widest <= 64) KV_NR(8);
    else if (widest <= 128) KV_NR(16);
    else if (widest <= 256) KV_NR(32);
    else KV_NR(64);
#undef KV_NR
    return (int)hipGetLastError();
  }
  const dim3 grid(T, (nh + 2 * nkv + 3) / 4);
  const size_t lds = (size_t)4 * dim * 4;
  if (f32) hipLaunchKernelGGL((norm_rope_write_kernel<float>), grid, dim3(256), lds, s, (const float*)proj, (float*)q, (float*)k_cache, (float*)v_cache, a);
  else hipLaunchKernelGGL((norm_rope_write_kernel<bf16raw>), grid, dim3(256), lds, s, (const bf16raw*)proj, (bf16raw*)q, (bf16raw*)k_cache, (bf16raw*)v_cache, a);
  return (int)hipGetLastError();
}

// bf16; q [T][nh][dvp + rt], cache [rows][dvp + rt]
int kvm_key_value_write(const void* proj, void* q, void* cache, float* key_scale, int rt, long long ldp, int q_off, int k_off, const float* bias, const float* q_norm, const float* k_norm,
                        const int* positions, const int* slots, const float* cos_t, const float* sin_t, int rot_dims, int T, int nh, int nkv, int dim, int dvp, int block_size, float eps, hipStream_t s) {
  if (T <= 0 || nh <= 0 || nkv <= 0 || nh % nkv || dim <= 0 || dim > 1024 || dvp < dim || rt < rot_dims || rot_dims < 0 || rot_dims > dim || (rot_dims & 1) || block_size <= 0 || !bias || !q_norm || !k_norm) return -1;
  const NormRopeArgs a{ldp, q_off, k_off, 0, bias, q_norm, k_norm, positions, slots, cos_t, sin_t, rot_dims, nh, nkv, dim, dim, dvp, dvp, block_size, eps};
  if (!((dim | dvp | rt | q_off | k_off) & 7) && !(rot_dims & 15) && !(ldp & 7) && !((uintptr_t)proj & 15) && dvp <= 512 && rt <= dvp) {
#define KV_KW(LPR) \
  hipLaunchKernelGGL((key_value_write_vec_kernel<LPR>), dim3(T, (nh + nkv + 256 / LPR - 1) / (256 / LPR)), dim3(256), 0, s, (const bf16raw*)proj, (bf16raw*)q, (bf16raw*)cache, key_scale, rt, a)
    if (dvp <= 64) KV_KW(8);
    else if (dvp <= 128) KV_KW(16);
    else if (dvp <= 256) KV_KW(32);
    else KV_KW(64);
#undef KV_KW
    return (int)hipGetLastError();
  }
  hipLaunchKernelGGL(key_value_write_kernel, dim3(T, (nh + nkv + 3) / 4), dim3(256), (size_t)4 * dim * 4, s, (const bf16raw*)proj, (bf16raw*)q, (bf16raw*)cache, key_scale, rt, a);
  return (int)hipGetLastError();
}

int kvm_row_attention(const void* q, int f32, const void* k_cache, const void* v_cache, const int* block_tables, int max_blocks, const int* tok_seq, const int* positions,
                      const int* slots, const void* gate, long long ld_gate, int gate_off, void* out, long long ldo, int o_off, int T, int nh, int nkv, int dkp, int vdim, int dvp,
                      int block_size, int chunk, int window, int keep, int gate_each, const float* sink, const float* rel, int rel_n, float scale, float out_scale, const int* row_flag, int only_flag,
                      hipStream_t s) {
  if (T <= 0 || nh <= 0 || nkv <= 0 || nh % nkv || (dkp & 3) || dkp > 1024 || vdim <= 0 || vdim > dvp || chunk < 0 || window < 0 || keep < 0 || (rel && rel_n < 1) || (only_flag >= 0 && !row_flag)) return -1;
  const RowAttentionArgs a{block_tables, max_blocks, tok_seq, positions, slots, nh, nkv, dkp, vdim, dvp, block_size, chunk, window, keep, sink, rel, rel_n, scale, out_scale, ld_gate, gate_off, gate == nullptr ? 0 : gate_each ? 2 : 1, ldo, o_off, only_flag, row_flag};
  return f32 ? launch_row_attention<float>(q, k_cache, v_cache, gate, out, T, a, s) : launch_row_attention<bf16raw>(q, k_cache, v_cache, gate, out, T, a, s);
}

// cache: [slots][rkp + rtp] (write 0: stays).  rot > 0: the query parts of nh heads go, rotated, to dst columns d_off + head d_head.
int kvm_latent_write(const void* proj, int f32, long long ldp, int c_off, const float* gain, const int* slots, const int* positions, void* cache, int write, int T, int rank, int rkp, int rot, int rtp,
                     int kr_off, const float* cos_t, const float* sin_t, int nh, int r_off, void* dst, long long ldd, int d_off, int d_head, float eps, hipStream_t s) {
  if (T <= 0 || rank <= 0 || rkp < rank || (rkp & 3) || rkp > 1024 || (write && ((c_off & 3) || !gain)) || (ldp & 3) || rot < 0 || (rot & 1) || (rtp & 3) || rtp < rot ||
      (rot && (!positions || !cos_t || !sin_t || nh <= 0 || !dst || d_head < rtp)))
    return -1;
  const LatentWriteArgs a{ldp, c_off, gain, slots, positions, T, rank, rkp, write, rot, rtp, kr_off, cos_t, sin_t, nh, r_off, ldd, d_off, d_head, eps};
  const dim3 grid((T + 3) / 4, rot ? 2 : 1);
  if (f32) hipLaunchKernelGGL((latent_write_kernel<float>), grid, dim3(256), 0, s, (const float*)proj, (float*)cache, (float*)dst, a);
  else hipLaunchKernelGGL((latent_write_kernel<bf16raw>), grid, dim3(256), 0, s, (const bf16raw*)proj, (bf16raw*)cache, (bf16raw*)dst, a);
  return (int)hipGetLastError();
}

// y: rows of ld columns (slabs or weighted rows as in kvm_gated_residual) or null; y2 with gate2 [T] or null; start: fp32 [T][ld] or null
int kvm_hyper_residual(float* x, int streams, void* xb, int f32, const void* y, long long y_ld, long long y_stride, int y_slabs, const float* y_weights, const void* y2, long long y2_ld,
                       long long y2_stride, int y2_slabs, const float* gate2, const float* mix, const float* out, const float* read, const float* next_g, const float* start, float eps, int T, int H,
                       int ld, hipStream_t s) {
  if (T <= 0 || H <= 0 || ld < H || (ld & 3) || ld > 32768 || streams < 1 || streams > 16 || !read || !next_g || (y && (!mix || !out || (y_ld & 3))) || (y_weights && y_slabs < 1) ||
      (y2 && (!y || !gate2 || (y2_ld & 3))) || (start && y))
    return -1;
  const RowSource ys{y, y_ld, y_stride, y_slabs, y_weights}, y2s{y2, y2_ld, y2_stride, y2_slabs, nullptr};
  const HyperArgs a{streams, mix, out, read, next_g, start, gate2, eps, H, ld};
  const size_t lds = (size_t)ld * 4;
#define KV_HR(Tt, NT, NS, EX)                                                                                                                                                \
  do {                                                                                                                                                                       \
    if (lds > 65536 && hipFuncSetAttribute((const void*)hyper_residual_kernel<Tt, NT, NS, EX>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) return -1; \
    hipLaunchKernelGGL((hyper_residual_kernel<Tt, NT, NS, EX>), dim3(T), dim3(NT), lds, s, x, (Tt*)xb, ys, y2s, a);                                                            \
  } while (0)
#define KV_HRS(Tt, NT)                          \
  do {                                          \
    if (streams == 1) KV_HR(Tt, NT, 1, true);   \
    else if (streams == 2) KV_HR(Tt, NT, 2, true); \
    else if (streams == 3) KV_HR(Tt, NT, 3, true); \
    else if (streams == 4) KV_HR(Tt, NT, 4, true); \
    else KV_HR(Tt, NT, 16, false);              \
  } while (0)
  if (ld <= 1024) { if (f32) KV_HRS(float, 256); else KV_HRS(bf16raw, 256); }
  else if (T <= 128 && streams <= 4) { if (f32) KV_HRS(float, 1024); else KV_HRS(bf16raw, 1024); }
  else { if (f32) KV_HRS(float, 512); else KV_HRS(bf16raw, 512); }
#undef KV_HRS
#undef KV_HR
  return (int)hipGetLastError();
}

// y, y2, y3: rows of ld columns (slabs or, y2, weighted rows as in kvm_gated_residual) or null
int kvm_parallel_residual(float* x, void* xb, void* xb2, int f32, const void* y, long long y_ld, long long y_stride, int y_slabs, const void* y2, long long y2_ld, int top, const float* y2_weights,
                          const void* y3, long long y3_ld, long long y3_stride, int y3_slabs, const float* bias, const float* g, const float* g2, float eps, int T, int H, int ld, hipStream_t s) {
  if (T <= 0 || H <= 0 || ld < H || (ld & 3) || ld > 32768 || !g || (g2 && !xb2) || ((y_ld | y2_ld | y3_ld) & 3) || (y2 && (!y2_weights || top < 1))) return -1;
  const RowSource ys{y, y_ld, y_stride, y_slabs, nullptr}, y2s{y2, y2_ld, 0, top, y2_weights}, y3s{y3, y3_ld, y3_stride, y3_slabs, nullptr};
  const ParallelArgs a{bias, g, g2, eps, H, ld};
  const size_t lds = (size_t)ld * 4;
#define KV_PR(Tt, NT)                                                                                                                                                \
  do {                                                                                                                                                               \
    if (lds > 65536 && hipFuncSetAttribute((const void*)parallel_residual_kernel<Tt, NT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) return -1; \
    hipLaunchKernelGGL((parallel_residual_kernel<Tt, NT>), dim3(T), dim3(NT), lds, s, x, (Tt*)xb, (Tt*)xb2, ys, y2s, y3s, a);                                          \
  } while (0)
  if (ld <= 1024) { if (f32) KV_PR(float, 256); else KV_PR(bf16raw, 256); }
  else if (T <= 128) { if (f32) KV_PR(float, 1024); else KV_PR(bf16raw, 1024); }  // few rows: the whole row at once
  else { if (f32) KV_PR(float, 512); else KV_PR(bf16raw, 512); }
#undef KV_PR
  return (int)hipGetLastError();
}

int kvm_softcap(void* x, int f32, long long stride, int S, int V, float cap, hipStream_t s) {
  if (S <= 0 || S > 65535 || V <= 0 || !(cap > 0.f)) return -1;
  const dim3 grid((V + 255) / 256, S);
  if (f32) hipLaunchKernelGGL((softcap_kernel<float>), grid, dim3(256), 0, s, (float*)x, stride, V, cap, 1.f / cap);
  else hipLaunchKernelGGL((softcap_kernel<bf16raw>), grid, dim3(256), 0, s, (bf16raw*)x, stride, V, cap, 1.f / cap);
  return (int)hipGetLastError();
}

int kvm_head_rows(const void* x, int f32, long long ldx, int x_off, int x_head, const void* w, int nh, int N, int K, int n_true, const void* gate, long long ld_gate, int gate_off, int gate_each, void* out,
                  long long ldo, int o_off, int o_head, float out_scale, const int* slots, int T, hipStream_t s) {
  if (T <= 0 || nh <= 0 || N <= 0 || K <= 0 || K > 8192 || n_true <= 0 || n_true > N) return -1;
  const HeadRowsArgs a{ldx, x_off, x_head, ldo, o_off, o_head, ld_gate, gate_off, gate == nullptr ? 0 : gate_each ? 2 : 1, N, K, n_true, out_scale, slots};
  const size_t lds = (size_t)K * 4;
  if (f32) hipLaunchKernelGGL((head_rows_kernel<float>), dim3(T, nh), dim3(256), lds, s, (const float*)x, (const float*)w, (const float*)gate, (float*)out, a);
  else hipLaunchKernelGGL((head_rows_kernel<bf16raw>), dim3(T, nh), dim3(256), lds, s, (const bf16raw*)x, (const bf16raw*)w, (const bf16raw*)gate, (bf16raw*)out, a);
  return (int)hipGetLastError();
}

int kvm_argmax_f32(const float* logits, long long stride, int S, int V, long long* out, hipStream_t s) {
  if (S <= 0 || V <= 0) return -1;
  hipLaunchKernelGGL(argmax_f32_kernel, dim3(S), dim3(1024), 0, s, logits, stride, V, out);
  return (int)hipGetLastError();
}

}  // extern "C"
