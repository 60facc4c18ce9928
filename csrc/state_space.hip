// Selective state space (state-space duality) for gfx950: linear attention whose decay and step size per head come from the token.  Per
// head h of group g, with the 32-bit state S [dim, vdim]:
//     dt = softplus(dt_raw + dt_bias),   S <- exp(-exp(A) dt) S + dt b x^T,   y = S^T c + D x;
// x (per head), b and c (per group) come out of a short causal convolution with bias and silu behind it.  The concatenated y is gated with
// silu(z) element by element, then divided in equal parts by their own root mean squares, with a gain per channel.  Steps, decays, state,
// scores and sums are fp32; T is the type of the projections, of the convolution's results and of the output.  Products: on the fp32 matrix
// instructions, or, for T = bf16 and sizes in eights, on the bf16 ones without losing anything: b, c and x are bf16 as they are, and the
// other operand (state, weighted scores, weighted x) is cut into three bf16 numbers, eight bits each, whose sum it is.
//
//   space_step_kernel   single tokens: convolution, step, state update and read-out.  A workgroup owns one head's state, every byte of which
//                       is read and written once, in whole rows.
//   Portions of several tokens, in chunks of 64 (counted from the portion's start):
//   space_conv_kernel   convolution, step sizes and logarithms of the decays, for all tokens in parallel
//   space_state_kernel  what a chunk adds to the state, sum_j decay(j -> end) dt_j b_j x_j^T, and its whole decay, all chunks and heads at once
//   space_scan_kernel   the chunks of a portion one after the other, element by element: each chunk's contribution is replaced by the state
//                       in front of it, the last state is kept; also the convolution inputs the next portion needs
//   space_out_kernel    y_i = decay(start -> i) S^T c_i + sum_{j<=i} decay(j -> i) dt_j (b_j . c_i) x_j + D x_i, all chunks and heads at once
//   space_state16_kernel, space_out16_kernel   these two on the bf16 matrix instructions
//   space_gate_kernel   gate and norms
//
// Decays inside a chunk are exponentials of differences of running sums, which are kept as sums of two floats.
// State: fp32 [slots][heads][dimp][dvp], sizes rounded up to 16 (what is behind dim / vdim stays zero); the convolution's last inputs, T
// [slots][taps][channels], position p at p % taps.  A portion that starts at position 0 takes both as zero, so nothing has to be cleared
// when a slot changes hands.  Channels are ordered x [heads vdim], b [groups dim], c [groups dim].

#include "attn_tiles.h"

struct KvsArgs {
  long long ldp; int z_off, x_off, dt_off;
  const float *conv_w, *conv_b, *dt_bias, *a_log, *skip, *norm;  // conv_w [taps][channels]
  int heads, groups, dim, vdim, dimp, dvp, taps, channels, norm_groups;
  float eps, out_scale;
  float* state;
  const int *tok_seq, *positions, *tok_kind, *tok_off;
  long long ldo; int o_off;
};

namespace {
using namespace elem;
using namespace attn;

constexpr int CHUNK = 64;
typedef __attribute__((ext_vector_type(4))) float f4;

template <typename T> __device__ inline float rounded(float v);
template <> __device__ inline float rounded<float>(float v) { return v; }
template <> __device__ inline float rounded<bf16raw>(float v) { return bf2f(f2bf(v)); }

// convolution and silu of channel c at row t, in T's precision; `back` = rows of the same portion in front of t
template <typename T>
__device__ inline float conv_silu(const KvsArgs& a, const T* __restrict__ proj, const T* __restrict__ ring, long long t, int pos, int back, int slot, int c) {
  const T* p = proj + t * a.ldp + a.x_off + c;
  float y = a.conv_b[c] + a.conv_w[(a.taps - 1) * a.channels + c] * ld(p);
#pragma unroll 4
  for (int j = 1; j < a.taps; ++j) {
    const T* src = j <= back ? p - j * a.ldp : ring + ((long long)slot * a.taps + (j <= pos ? pos - j : 0) % a.taps) * a.channels + c;
    const float x = ld(src);
    y += a.conv_w[(a.taps - 1 - j) * a.channels + c] * (j <= pos ? x : 0.f);
  }
  return rounded<T>(silu(y));
}

__device__ inline float step_size(const KvsArgs& a, float raw, int h) { return softplus(raw + a.dt_bias[h]); }
__device__ inline float log2_decay(const KvsArgs& a, float dt, int h) { return -1.4426950408889634f * fast_exp(a.a_log[h]) * dt; }

// ---- single tokens: grid (listed rows, heads); thread = a group of state rows x 4 columns
template <typename T>
__global__ __launch_bounds__(256) void space_step_kernel(const T* __restrict__ proj, T* __restrict__ ring, float* __restrict__ y, const int* __restrict__ rows, KvsArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const long long t = rows[blockIdx.x];
  const int h = blockIdx.y, tid = threadIdx.x;
  if (t < 0 || a.tok_kind[t] != 1) return;  // unused entry, or a padding row
  const int pos = a.positions[t], slot = a.tok_seq[t];
  const int rep = a.heads / a.groups, g = h / rep, inner = a.heads * a.vdim;
  const int nc = a.dvp >> 2, nrg = 256 / nc;
  const int rg = tid / nc, col = (tid - rg * nc) * 4;
  const bool on = rg < nrg;
  float* bs = sm;              // [dimp]: dt b
  float* cs = bs + a.dimp;     // [dimp]
  float* xs = cs + a.dimp;     // [dvp]
  float* red = xs + a.dvp;     // [nrg][dvp]
  float* st = a.state + ((long long)slot * a.heads + h) * a.dimp * a.dvp + col;
  constexpr int U = 8;
  float4 s[U];
  auto fetch = [&](int r0) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int r = r0 + u * nrg;
      s[u] = on && r < a.dimp && pos > 0 ? ld4(st + (long long)r * a.dvp) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
  };
  fetch(rg);
  const float dt = step_size(a, ld(proj + t * a.ldp + a.dt_off + h), h);
  const float decay = __builtin_amdgcn_exp2f(log2_decay(a, dt, h));
  const int b0 = inner + g * a.dim, c0 = b0 + a.groups * a.dim;
  for (int i = tid; i < 2 * a.dimp + a.dvp; i += 256) {
    const int which = i < a.dimp ? 0 : i < 2 * a.dimp ? 1 : 2, d = i - which * a.dimp;
    float v = 0.f;
    if (d < (which == 2 ? a.vdim : a.dim)) v = conv_silu<T>(a, proj, ring, t, pos, 0, slot, (which == 0 ? b0 : which == 1 ? c0 : h * a.vdim) + d);
    sm[i] = which == 0 ? v * dt : v;
  }
  __syncthreads();
  const float4 x = on ? ld4(xs + col) : make_float4(0.f, 0.f, 0.f, 0.f);
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
  for (int r0 = rg; r0 < a.dimp; r0 += U * nrg) {
    if (r0 != rg) fetch(r0);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int r = r0 + u * nrg;
      if (on && r < a.dimp) {
        const float b = bs[r], c = cs[r];
        s[u].x = s[u].x * decay + b * x.x; s[u].y = s[u].y * decay + b * x.y; s[u].z = s[u].z * decay + b * x.z; s[u].w = s[u].w * decay + b * x.w;
        o.x += c * s[u].x; o.y += c * s[u].y; o.z += c * s[u].z; o.w += c * s[u].w;
        st4(st + (long long)r * a.dvp, s[u]);
      }
    }
  }
  if (on) st4(red + rg * a.dvp + col, o);
  __syncthreads();
  for (int d = tid; d < a.vdim; d += 256) {
    float v = a.skip[h] * xs[d];
    for (int r = 0; r < nrg; ++r) v += red[r * a.dvp + d];
    y[t * inner + h * a.vdim + d] = v;
  }
  // the ring entry of this position was last used for position pos - taps, which nobody reads any more
  T* rw = ring + ((long long)slot * a.taps + pos % a.taps) * a.channels;
  const T* pr = proj + t * a.ldp + a.x_off;
  for (int d = tid; d < a.vdim; d += 256) rw[h * a.vdim + d] = pr[h * a.vdim + d];
  if (h % rep == 0)
    for (int d = tid; d < a.dim; d += 256) {
      rw[b0 + d] = pr[b0 + d];
      rw[c0 + d] = pr[c0 + d];
    }
}

// ---- portions: convolution of all channels (VEC per thread, RUN tokens one after the other); the last row of workgroups: steps and decays.
// xbc T [rows][channels]; dts, las fp32 [heads][rows]
constexpr int RUN = 8;

template <typename T, int VEC, int TAPS>
__global__ __launch_bounds__(256) void space_conv_kernel(const T* __restrict__ proj, const T* __restrict__ ring, T* __restrict__ xbc, float* __restrict__ dts, float* __restrict__ las, int n_rows,
                                                         KvsArgs a) {
  const int t0 = blockIdx.x * RUN, t1 = t0 + RUN < n_rows ? t0 + RUN : n_rows;
  if (blockIdx.y == gridDim.y - 1) {
    for (int i = threadIdx.x; i < a.heads * (t1 - t0); i += 256) {
      const int h = i / (t1 - t0);
      const long long t = t0 + i - h * (t1 - t0);
      if (a.tok_kind[t] != 2) continue;
      const float dt = step_size(a, ld(proj + t * a.ldp + a.dt_off + h), h);
      dts[(long long)h * n_rows + t] = dt;
      las[(long long)h * n_rows + t] = log2_decay(a, dt, h);
    }
    return;
  }
  const int c = (blockIdx.y * 256 + threadIdx.x) * VEC;
  if (c >= a.channels) return;
  if constexpr (VEC == 1) {
    for (long long t = t0; t < t1; ++t)
      if (a.tok_kind[t] == 2) st(xbc + t * a.channels + c, conv_silu<T>(a, proj, ring, t, a.positions[t], a.tok_off[t], a.tok_seq[t], c));
  } else {
    static_assert(sizeof(T) == 2 && VEC == 8, "16-byte pieces of bf16");
    typedef __attribute__((ext_vector_type(8))) unsigned short piece;
    const int taps = TAPS ? TAPS : a.taps;
    float bias[VEC], w[TAPS ? TAPS : 1][VEC];
    auto load8 = [](float* d, const float* p) { *reinterpret_cast<float4*>(d) = ld4(p); *reinterpret_cast<float4*>(d + 4) = ld4(p + 4); };
    load8(bias, a.conv_b + c);
    if constexpr (TAPS > 0) {
#pragma unroll
      for (int j = 0; j < TAPS; ++j) load8(w[j], a.conv_w + (taps - 1 - j) * a.channels + c);  // w[j]: of the input j tokens back
    }
    const T* p0 = proj + a.x_off + c;
    auto input = [&](long long t, int j, int pos, int back, int slot) __attribute__((always_inline)) {  // (before the sequence's start: nothing)
      piece v = (piece)(unsigned short)0;
      if (j <= pos) v = *reinterpret_cast<const piece*>(j <= back ? p0 + (t - j) * a.ldp : ring + ((long long)slot * taps + (pos - j) % taps) * a.channels + c);
      return v;
    };
    piece in[TAPS ? TAPS : 1];  // in[j]: the input j tokens back
    for (long long t = t0; t < t1; ++t) {
      if (a.tok_kind[t] != 2) continue;
      const int pos = a.positions[t], back = a.tok_off[t], slot = a.tok_seq[t];
      float s[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) s[e] = bias[e];
      if constexpr (TAPS > 0) {
        const bool next = t > t0 && back > 0;  // (the row in front is the token in front: its window moves on)
#pragma unroll
        for (int j = TAPS - 1; j > 0; --j) in[j] = next ? in[j - 1] : input(t, j, pos, back, slot);
        in[0] = input(t, 0, pos, back, slot);
#pragma unroll
        for (int j = 0; j < TAPS; ++j)
#pragma unroll
          for (int e = 0; e < VEC; ++e) s[e] += w[j][e] * bf2f(in[j][e]);
      } else {
        for (int j = 0; j < taps; ++j) {
          const piece v = input(t, j, pos, back, slot);
          float wv[VEC];
          load8(wv, a.conv_w + (taps - 1 - j) * a.channels + c);
#pragma unroll
          for (int e = 0; e < VEC; ++e) s[e] += wv[e] * bf2f(v[e]);
        }
      }
      piece o;
#pragma unroll
      for (int e = 0; e < VEC; ++e) o[e] = f2bf(silu(s[e]));
      *reinterpret_cast<piece*>(xbc + t * a.channels + c) = o;
    }
  }
}

// four consecutive of n entries from d on, zero behind them; vec: n and the address are multiples of four
template <typename T>
__device__ inline float4 four(const T* p, int d, int n, bool vec) {
  if (vec) {  // (no branches: many of these are in flight at a time)
    const float4 v = ld4(p + (d < n ? d : n - 4));
    return d < n ? v : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
  if (d < n) v.x = ld(p + d);
  if (d + 1 < n) v.y = ld(p + d + 1);
  if (d + 2 < n) v.z = ld(p + d + 2);
  if (d + 3 < n) v.w = ld(p + d + 3);
  return v;
}

// running sums of a chunk's decay logarithms, as sums of two floats (one wave; entries behind the chunk repeat the last)
__device__ inline void running_sums(const float* __restrict__ las, int n, float* hi, float* lo) {
  const int lane = threadIdx.x & 63;
  double v = lane < n ? (double)las[lane] : 0.0;
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const double u = __shfl_up(v, o, 64);
    if (lane >= o) v += u;
  }
  const float f = (float)v;
  hi[lane] = f;
  lo[lane] = (float)(v - (double)f);
}

struct SpaceChunks { const int* row; const int* n; int n_rows; const float* dts; const float* las; };

// ---- a chunk's contribution to the state: grid (heads, chunks, blocks of DB x VB); 4 waves, a quarter of the block each
template <typename T, int DB, int VB>
__global__ __launch_bounds__(256) void space_state_kernel(const T* __restrict__ xbc, float* __restrict__ ws, float* __restrict__ whole, SpaceChunks c, int v_blocks, KvsArgs a) {
  constexpr int KS = DB + 16, VS = VB + 16;  // (a fragment's four rows lie in different banks)
  constexpr int ND = DB / 32, NV = VB / 32;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float hi[CHUNK], lo[CHUNK];
  float* k_s = sm;               // [CHUNK][KS]
  float* v_s = sm + CHUNK * KS;  // [CHUNK][VS]
  const int h = blockIdx.x, b = blockIdx.y;
  const int n = c.n[b];
  if (n <= 0) return;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, lr = lane & 15, lq = lane >> 4;
  const int d_blk = blockIdx.z / v_blocks * DB, v_blk = blockIdx.z % v_blocks * VB;
  const long long row0 = c.row[b];
  const int g = h / (a.heads / a.groups), inner = a.heads * a.vdim;
  const bool vec = !((a.dim | a.channels | inner) & 3), v_vec = !((a.vdim | a.channels) & 3);
  const float* dts = c.dts + (long long)h * c.n_rows + row0;
  if (wave == 0) running_sums(c.las + (long long)h * c.n_rows + row0, n, hi, lo);
  const int rows = (n + 3) & ~3;
#pragma unroll 4
  for (int i = tid; i < rows * (VB / 4); i += 256) {
    const int j = i / (VB / 4), d = i % (VB / 4) * 4;
    const T* p = xbc + (row0 + (j < n ? j : n - 1)) * a.channels + h * a.vdim;  // (rows past the last one: weight zero)
    st4(v_s + j * VS + d, four(p, v_blk + d, a.vdim, v_vec));
  }
  __syncthreads();
  if (blockIdx.z == 0 && tid == 0) whole[(long long)b * a.heads + h] = __builtin_amdgcn_exp2f(hi[n - 1] + lo[n - 1]);
#pragma unroll 4
  for (int i = tid; i < rows * (DB / 4); i += 256) {
    const int j = i / (DB / 4), d = i % (DB / 4) * 4;
    const int jr = j < n ? j : n - 1;
    float4 k = four(xbc + (row0 + jr) * a.channels + inner + g * a.dim, d_blk + d, a.dim, vec);
    const float f = j < n ? dts[jr] * __builtin_amdgcn_exp2f((hi[n - 1] - hi[jr]) + (lo[n - 1] - lo[jr])) : 0.f;
    k.x *= f; k.y *= f; k.z *= f; k.w *= f;
    st4(k_s + j * KS + d, k);
  }
  __syncthreads();
  const int d0 = (wave >> 1) * (DB / 2), v0 = (wave & 1) * (VB / 2);
  f4 acc[ND][NV];
#pragma unroll
  for (int x = 0; x < ND; ++x)
#pragma unroll
    for (int y = 0; y < NV; ++y) acc[x][y] = (f4){0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int j = 0; j < rows; j += 4) {
    float ka[ND], vb[NV];
#pragma unroll
    for (int x = 0; x < ND; ++x) ka[x] = k_s[(j + lq) * KS + d0 + 16 * x + lr];
#pragma unroll
    for (int y = 0; y < NV; ++y) vb[y] = v_s[(j + lq) * VS + v0 + 16 * y + lr];
#pragma unroll
    for (int x = 0; x < ND; ++x)
#pragma unroll
      for (int y = 0; y < NV; ++y) acc[x][y] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[x], vb[y], acc[x][y], 0, 0, 0);
  }
  float* u = ws + ((long long)b * a.heads + h) * a.dimp * a.dvp;
#pragma unroll
  for (int x = 0; x < ND; ++x)
#pragma unroll
    for (int y = 0; y < NV; ++y) {
      const int d = d_blk + d0 + 16 * x, v = v_blk + v0 + 16 * y;  // (whole tiles are inside or outside)
      if (d >= a.dimp || v >= a.dvp) continue;
#pragma unroll
      for (int e = 0; e < 4; ++e) u[(long long)(d + 4 * lq + e) * a.dvp + v + lr] = acc[x][y][e];
    }
}

// ---- the same on the bf16 matrix instructions (sizes in eights): grid (heads, chunks, blocks of 128 x 64); wave: 64 x 32 of a block.  b and
// the three parts of the weighted x lie in LDS as they come, rows of a token; both operands are transposed reads, whose order of the
// tokens is the same.
typedef __attribute__((ext_vector_type(8))) unsigned short us8;

// v as the sum of three bf16 numbers (the first eight bits, the next eight, the rest)
__device__ inline void cut3(float v, bf16raw& a, bf16raw& b, bf16raw& c) {
  const unsigned int h = __float_as_uint(v) & 0xffff0000u;
  const float r = v - __uint_as_float(h);
  const unsigned int m = __float_as_uint(r) & 0xffff0000u;
  a = (bf16raw)(h >> 16);
  b = (bf16raw)(m >> 16);
  c = (bf16raw)(__float_as_uint(r - __uint_as_float(m)) >> 16);
}

// rows base + 4 lq .. + 3 and base + 16 + 4 lq .. + 3 of column 16 n + lr of an image [rows][D] swizzled by kv_swz
template <int D>
__device__ inline frag_ab token_pair(const bf16raw* img, int base, int n) {
  const int lane = threadIdx.x & 63, lr = lane & 15, lq = lane >> 4;
  const int r = base + 4 * lq + (lr >> 2), c = 2 * n + ((lr & 3) >> 1), o = (lr & 1) * 4;
  const struct { tr_b64 lo, hi; } v = {__builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_tr_b64*)(img + r * D + ((c ^ kv_swz<D>(r)) << 3) + o)),
                                       __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_tr_b64*)(img + (r + 16) * D + ((c ^ kv_swz<D>(r + 16)) << 3) + o))};
  return __builtin_bit_cast(frag_ab, v);
}

// columns first .. first + D - 1 (of n) of a chunk's rows, into an image swizzled by kv_swz; zero behind the columns and behind the rows
template <int D>
__device__ inline void stage_rows(bf16raw* img, const bf16raw* __restrict__ src, long long ld, int rows, int first, int n) {
#pragma unroll
  for (int it = 0; it < CHUNK * (D / 8) / 256; ++it) {
    const int i = threadIdx.x + it * 256, j = i / (D / 8), c = i % (D / 8), d = first + 8 * c;
    us8 v = *reinterpret_cast<const us8*>(src + (long long)(j < rows ? j : rows - 1) * ld + (d < n ? d : 0));
    if (j >= rows || d >= n) v = (us8)(unsigned short)0;
    *reinterpret_cast<us8*>(img + j * D + ((c ^ kv_swz<D>(j)) << 3)) = v;
  }
}

__global__ __launch_bounds__(256, 3) void space_state16_kernel(const bf16raw* __restrict__ xbc, float* __restrict__ ws, float* __restrict__ whole, SpaceChunks c, int v_blocks, KvsArgs a) {
  __shared__ __attribute__((aligned(16))) bf16raw b_s[CHUNK * 128], x_s[3][CHUNK * 64];
  __shared__ float hi[CHUNK], lo[CHUNK];
  const int h = blockIdx.x, b = blockIdx.y;
  const int n = c.n[b];
  if (n <= 0) return;
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, lr = lane & 15, lq = lane >> 4;
  const int d_blk = blockIdx.z / v_blocks * 128, v_blk = blockIdx.z % v_blocks * 64;
  const long long row0 = c.row[b];
  const int g = h / (a.heads / a.groups), inner = a.heads * a.vdim;
  const bf16raw* rows = xbc + row0 * a.channels;
  us8 x[2];  // two pieces of the block of x: on their way while the decays are summed
#pragma unroll
  for (int it = 0; it < 2; ++it) {
    const int i = tid + it * 256, j = i >> 3, d = v_blk + 8 * (i & 7);
    x[it] = *reinterpret_cast<const us8*>(rows + (long long)(j < n ? j : n - 1) * a.channels + h * a.vdim + (d < a.vdim ? d : 0));
    if (d >= a.vdim) x[it] = (us8)(unsigned short)0;
  }
  stage_rows<128>(b_s, rows + inner + g * a.dim, a.channels, n, d_blk, a.dim);
  if (wave == 0) running_sums(c.las + (long long)h * c.n_rows + row0, n, hi, lo);
  __syncthreads();
  if (blockIdx.z == 0 && tid == 0) whole[(long long)b * a.heads + h] = __builtin_amdgcn_exp2f(hi[n - 1] + lo[n - 1]);
#pragma unroll
  for (int it = 0; it < 2; ++it) {
    const int i = tid + it * 256, j = i >> 3, ch = i & 7;
    const float f = j < n ? c.dts[(long long)h * c.n_rows + row0 + j] * __builtin_amdgcn_exp2f((hi[n - 1] - hi[j]) + (lo[n - 1] - lo[j])) : 0.f;
    us8 p[3];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      bf16raw q0, q1, q2;
      cut3(f * bf2f(x[it][e]), q0, q1, q2);
      p[0][e] = q0; p[1][e] = q1; p[2][e] = q2;
    }
#pragma unroll
    for (int k = 0; k < 3; ++k) *reinterpret_cast<us8*>(&x_s[k][j * 64 + ((ch ^ kv_swz<64>(j)) << 3)]) = p[k];
  }
  __syncthreads();
  const int d0 = (wave >> 1) * 64, v0 = (wave & 1) * 32;
  if (d_blk + d0 >= a.dimp) return;
  frag_acc4 acc[4][2];
#pragma unroll
  for (int x_ = 0; x_ < 4; ++x_)
#pragma unroll
    for (int y = 0; y < 2; ++y) acc[x_][y] = (frag_acc4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < CHUNK; j += 32) {
    frag_ab ba[4], xb[2][3];
#pragma unroll
    for (int x_ = 0; x_ < 4; ++x_) ba[x_] = token_pair<128>(b_s, j, d0 / 16 + x_);
#pragma unroll
    for (int y = 0; y < 2; ++y)
#pragma unroll
      for (int k = 0; k < 3; ++k) xb[y][k] = token_pair<64>(x_s[k], j, v0 / 16 + y);
#pragma unroll
    for (int k = 2; k >= 0; --k)  // (the small parts first)
#pragma unroll
      for (int x_ = 0; x_ < 4; ++x_)
#pragma unroll
        for (int y = 0; y < 2; ++y) acc[x_][y] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ba[x_], xb[y][k], acc[x_][y], 0, 0, 0);
  }
  float* u = ws + ((long long)b * a.heads + h) * a.dimp * a.dvp;
#pragma unroll
  for (int x_ = 0; x_ < 4; ++x_)
#pragma unroll
    for (int y = 0; y < 2; ++y) {
      const int d = d_blk + d0 + 16 * x_, v = v_blk + v0 + 16 * y;  // (whole tiles are inside or outside)
      if (d >= a.dimp || v >= a.dvp) continue;
#pragma unroll
      for (int e = 0; e < 4; ++e) u[(long long)(d + 4 * lq + e) * a.dvp + v + lr] = acc[x_][y][e];
    }
}

// ---- portions: grid (elements / 1024, heads + 1, portions), four elements per thread; the workgroups behind the heads keep the last inputs
template <typename T>
__global__ __launch_bounds__(256) void space_scan_kernel(const T* __restrict__ proj, T* __restrict__ ring, float* __restrict__ ws, const float* __restrict__ whole, const int* __restrict__ seg_row,
                                                         const int* __restrict__ seg_n, const int* __restrict__ seg_pos, const int* __restrict__ seg_slot, const int* __restrict__ first_chunk,
                                                         int n_chunks, KvsArgs a) {
  const int h = blockIdx.y, sg = blockIdx.z;
  const int n = seg_n[sg];
  if (n < 2) return;
  if (h == a.heads) {
    const int keep = n < a.taps ? n : a.taps;
    for (int c = blockIdx.x * 256 + threadIdx.x; c < a.channels; c += gridDim.x * 256)
      for (int i = n - keep; i < n; ++i)
        ring[((long long)seg_slot[sg] * a.taps + (seg_pos[sg] + i) % a.taps) * a.channels + c] = proj[(long long)(seg_row[sg] + i) * a.ldp + a.x_off + c];
    return;
  }
  const int size = a.dimp * a.dvp, i = (blockIdx.x * 256 + threadIdx.x) * 4;
  const int c0 = first_chunk[sg], nc = (n + CHUNK - 1) / CHUNK;
  if (i >= size || c0 < 0 || c0 + nc > n_chunks) return;
  float* st = a.state + ((long long)seg_slot[sg] * a.heads + h) * size + i;
  float* u = ws + ((long long)c0 * a.heads + h) * size + i;
  const float* f = whole + (long long)c0 * a.heads + h;
  const long long step = (long long)a.heads * size;
  float4 s = seg_pos[sg] > 0 ? ld4(st) : make_float4(0.f, 0.f, 0.f, 0.f);
  constexpr int U = 4;  // chunks in flight
  for (int c = 0; c < nc; c += U) {
    float4 x[U];
    float d[U];
#pragma unroll
    for (int e = 0; e < U; ++e) {
      x[e] = c + e < nc ? ld4(u + (c + e) * step) : make_float4(0.f, 0.f, 0.f, 0.f);
      d[e] = f[(long long)(c + e < nc ? c + e : nc - 1) * a.heads];
    }
#pragma unroll
    for (int e = 0; e < U; ++e) {
      if (c + e >= nc) break;
      st4(u + (c + e) * step, s);
      s.x = s.x * d[e] + x[e].x; s.y = s.y * d[e] + x[e].y; s.z = s.z * d[e] + x[e].z; s.w = s.w * d[e] + x[e].w;
    }
  }
  st4(st, s);
}

// ---- outputs: grid (heads, chunks, blocks of 64 NT columns).  The waves share the columns of y (NT tiles of 16 each), so the state and the
// inputs are read once per workgroup, straight from memory; b and c pass through LDS in blocks of 64 dimensions.
template <typename T, int NT>
__global__ __launch_bounds__(256, NT <= 2 ? 3 : 2) void space_out_kernel(const T* __restrict__ xbc, const float* __restrict__ ws, float* __restrict__ out, SpaceChunks c, KvsArgs a) {
  constexpr int S = CHUNK + 4;  // (16 rows x 4 entries of a fragment lie in different banks)
  __shared__ __attribute__((aligned(16))) float q_s[CHUNK * S], k_s[CHUNK * S], p_s[CHUNK * S];
  __shared__ float hi[CHUNK], lo[CHUNK], dt_s[CHUNK];
  const int h = blockIdx.x, b = blockIdx.y;
  const int n = c.n[b];
  if (n <= 0) return;
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, lr = lane & 15, lq = lane >> 4;
  const long long row0 = c.row[b];
  const int g = h / (a.heads / a.groups), inner = a.heads * a.vdim;
  const bool vec = !((a.dim | a.channels | inner) & 3);
  const int tiles = a.dvp / 16, tile0 = blockIdx.z * 4 * NT;
  const float* s_in = ws + ((long long)b * a.heads + h) * a.dimp * a.dvp;
  const int rts = (n + 15) >> 4;  // row tiles in use
  if (wave == 0) running_sums(c.las + (long long)h * c.n_rows + row0, n, hi, lo);
  else if (wave == 1) dt_s[lane] = c.dts[(long long)h * c.n_rows + row0 + (lane < n ? lane : n - 1)];
  f4 o[4][NT], p[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    p[r] = (f4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int y = 0; y < NT; ++y) o[r][y] = (f4){0.f, 0.f, 0.f, 0.f};
  }
  int col[NT], vcol[NT];  // the lane's columns (tiles past the last one: the last one again; vcol: the last column instead of those behind it)
  bool live[NT];
#pragma unroll
  for (int y = 0; y < NT; ++y) {
    const int tl = tile0 + wave * NT + y;
    col[y] = 16 * (tl < tiles ? tl : tiles - 1) + lr;
    vcol[y] = col[y] < a.vdim ? col[y] : a.vdim - 1;
    live[y] = tl < tiles && col[y] < a.vdim;
  }
  for (int db = 0; db < a.dimp; db += 64) {
    if (db) __syncthreads();
    const int nd = a.dimp - db < 64 ? a.dimp - db : 64;  // (a multiple of 16)
    float sb[16][NT];  // the block's rows of the state: on their way while b and c are
#pragma unroll
    for (int u = 0; u < 16; ++u)
#pragma unroll
      for (int y = 0; y < NT; ++y) sb[u][y] = s_in[(long long)(4 * u < nd ? db + 4 * u + lq : lq) * a.dvp + col[y]];
#pragma unroll 4
    for (int i = tid; i < CHUNK * 16; i += 256) {
      const int j = i >> 4, d = (i & 15) * 4;
      const T* pr = xbc + (row0 + (j < n ? j : n - 1)) * a.channels + inner + g * a.dim;  // (rows past the last one: it again, never used)
      st4(k_s + j * S + d, four(pr, db + d, a.dim, vec));
      st4(q_s + j * S + d, four(pr + a.groups * a.dim, db + d, a.dim, vec));
    }
    __syncthreads();
#pragma unroll
    for (int u = 0; u < 16; ++u) {
      if (4 * u >= nd) break;
      float qa[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) qa[r] = q_s[(16 * r + lr) * S + 4 * u + lq];
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int y = 0; y < NT; ++y) o[r][y] = __builtin_amdgcn_mfma_f32_16x16x4f32(qa[r], sb[u][y], o[r][y], 0, 0, 0);
    }
    if (wave < rts) {
#pragma unroll 4
      for (int d = 0; d < nd; d += 4) {
        const float q = q_s[(16 * wave + lr) * S + d + lq];
#pragma unroll
        for (int x = 0; x < 4; ++x)
          if (x <= wave) p[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(q, k_s[(16 * x + lr) * S + d + lq], p[x], 0, 0, 0);
      }
    }
  }
  float vb[16][NT];  // the inputs: on their way while the scores are weighted
#pragma unroll
  for (int u = 0; u < 16; ++u) {
    const int j = 4 * u + lq;
    const T* vp = xbc + (row0 + (j < n ? j : n - 1)) * a.channels + h * a.vdim;  // (rows past the last one have weight zero)
#pragma unroll
    for (int y = 0; y < NT; ++y) vb[u][y] = ld(vp + vcol[y]);
  }
  // scores of row tile `wave`, weighted; y so far, decayed
#pragma unroll
  for (int x = 0; x < 4; ++x)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = 16 * wave + 4 * lq + e, j = 16 * x + lr;
      p_s[i * S + j] = j <= i && i < n ? p[x][e] * dt_s[j] * __builtin_amdgcn_exp2f((hi[i] - hi[j]) + (lo[i] - lo[j])) : 0.f;
    }
#pragma unroll
  for (int r = 0; r < 4; ++r)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = 16 * r + 4 * lq + e;
      const float f = __builtin_amdgcn_exp2f(hi[i] + lo[i]);
#pragma unroll
      for (int y = 0; y < NT; ++y) o[r][y][e] *= f;
    }
  __syncthreads();
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
    if (jt >= rts) break;
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (r < jt) continue;
        const float pa = p_s[(16 * r + lr) * S + 16 * jt + 4 * u + lq];
#pragma unroll
        for (int y = 0; y < NT; ++y) o[r][y] = __builtin_amdgcn_mfma_f32_16x16x4f32(pa, vb[4 * jt + u][y], o[r][y], 0, 0, 0);
      }
  }
  const float skip = a.skip[h];
#pragma unroll
  for (int u = 0; u < 16; ++u) {
    const int i = 16 * (u >> 2) + 4 * lq + (u & 3);
    const long long row = row0 + (i < n ? i : n - 1);
#pragma unroll
    for (int y = 0; y < NT; ++y) {
      const float x = ld(xbc + row * a.channels + h * a.vdim + vcol[y]);
      if (i < n && live[y]) out[row * inner + h * a.vdim + col[y]] = o[u >> 2][y][u & 3] + skip * x;
    }
  }
}

// ---- the same on the bf16 matrix instructions (sizes in eights): grid (heads, chunks, blocks of 64 columns), a wave has 16 of the columns.
// c and b lie in LDS in blocks of 128 dimensions, later the three parts of the weighted scores in their place; the state comes straight
// from memory and is cut in registers; x is read transposed, and the scores' tokens in that order.
__global__ __launch_bounds__(256, 3) void space_out16_kernel(const bf16raw* __restrict__ xbc, const float* __restrict__ ws, float* __restrict__ out, SpaceChunks c, KvsArgs a) {
  constexpr int PS = CHUNK + 8;
  __shared__ __attribute__((aligned(16))) bf16raw cb_s[2][CHUNK * 128], x_s[CHUNK * 64];
  __shared__ float hi[CHUNK], lo[CHUNK], dt_s[CHUNK];
  static_assert(3 * CHUNK * PS <= 2 * CHUNK * 128, "the scores' parts lie where c and b were");
  bf16raw* c_s = cb_s[0];
  bf16raw* b_s = cb_s[1];
  bf16raw* p_s = cb_s[0];  // [3][CHUNK][PS]
  const int h = blockIdx.x, b = blockIdx.y;
  const int n = c.n[b];
  if (n <= 0) return;
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, lr = lane & 15, lq = lane >> 4;
  const long long row0 = c.row[b];
  const int g = h / (a.heads / a.groups), inner = a.heads * a.vdim, v_blk = blockIdx.z * 64;
  const bf16raw* rows = xbc + row0 * a.channels;
  const int col = v_blk + 16 * wave + lr, colc = col < a.dvp ? col : a.dvp - 1;
  const float* s_in = ws + ((long long)b * a.heads + h) * a.dimp * a.dvp + colc;
  const int rts = (n + 15) >> 4;  // row tiles in use
  frag_acc4 o[4], p[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) o[r] = p[r] = (frag_acc4){0.f, 0.f, 0.f, 0.f};
  for (int db = 0; db < a.dimp; db += 128) {
    float sb[4][8];  // the block's rows of the state (behind the last one: the last again, c is zero there)
#pragma unroll
    for (int k = 0; k < 4; ++k)
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int d = db + 32 * k + 8 * lq + e;
        sb[k][e] = s_in[(long long)(d < a.dimp ? d : a.dimp - 1) * a.dvp];
      }
    if (db) __syncthreads();
    stage_rows<128>(c_s, rows + inner + (a.groups + g) * a.dim, a.channels, n, db, a.dim);
    stage_rows<128>(b_s, rows + inner + g * a.dim, a.channels, n, db, a.dim);
    if (db == 0) {
      stage_rows<64>(x_s, rows + h * a.vdim, a.channels, n, v_blk, a.vdim);
      if (wave == 0) running_sums(c.las + (long long)h * c.n_rows + row0, n, hi, lo);
      else if (wave == 1) dt_s[lane] = c.dts[(long long)h * c.n_rows + row0 + (lane < n ? lane : n - 1)];
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      if (db + 32 * k >= a.dimp) break;
      us8 cut[3];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        bf16raw q0, q1, q2;
        cut3(sb[k][e], q0, q1, q2);
        cut[0][e] = q0; cut[1][e] = q1; cut[2][e] = q2;
      }
      frag_ab ca[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = 16 * r + lr;
        ca[r] = *reinterpret_cast<const frag_ab*>(&c_s[row * 128 + (((4 * k + lq) ^ kv_swz<128>(row)) << 3)]);
      }
#pragma unroll
      for (int q = 2; q >= 0; --q)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ca[r], __builtin_bit_cast(frag_ab, cut[q]), o[r], 0, 0, 0);
      if (wave < rts) {
        const int mine = 16 * wave + lr;
        const frag_ab cm = *reinterpret_cast<const frag_ab*>(&c_s[mine * 128 + (((4 * k + lq) ^ kv_swz<128>(mine)) << 3)]);
#pragma unroll
        for (int x = 0; x < 4; ++x)
          if (x <= wave) {
            const int row = 16 * x + lr;
            p[x] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cm, *reinterpret_cast<const frag_ab*>(&b_s[row * 128 + (((4 * k + lq) ^ kv_swz<128>(row)) << 3)]), p[x], 0, 0, 0);
          }
      }
    }
  }
  __syncthreads();  // (nobody reads c and b any more)
  // scores of row tile `wave`, weighted; y so far, decayed
#pragma unroll
  for (int x = 0; x < 4; ++x)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = 16 * wave + 4 * lq + e, j = 16 * x + lr;
      const float v = j <= i && i < n ? p[x][e] * dt_s[j] * __builtin_amdgcn_exp2f((hi[i] - hi[j]) + (lo[i] - lo[j])) : 0.f;
      bf16raw q0, q1, q2;
      cut3(v, q0, q1, q2);
      p_s[i * PS + j] = q0;
      p_s[(CHUNK + i) * PS + j] = q1;
      p_s[(2 * CHUNK + i) * PS + j] = q2;
    }
#pragma unroll
  for (int r = 0; r < 4; ++r)
#pragma unroll
    for (int e = 0; e < 4; ++e) o[r][e] *= __builtin_amdgcn_exp2f(hi[16 * r + 4 * lq + e] + lo[16 * r + 4 * lq + e]);
  __syncthreads();
#pragma unroll
  for (int j = 0; j < CHUNK; j += 32) {
    if (j >= n) break;
    const frag_ab xv = token_pair<64>(x_s, j, wave);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if (16 * r + 15 < j) continue;
#pragma unroll
      for (int q = 2; q >= 0; --q) {
        const bf16raw* pp = p_s + (q * CHUNK + 16 * r + lr) * PS + j + 4 * lq;
        const struct { frag_b64 lo, hi; } pa = {*reinterpret_cast<const frag_b64*>(pp), *reinterpret_cast<const frag_b64*>(pp + 16)};
        o[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(frag_ab, pa), xv, o[r], 0, 0, 0);
      }
    }
  }
  if (col >= a.vdim) return;
  const float skip = a.skip[h];
  const int cx = 16 * wave + lr;
#pragma unroll
  for (int r = 0; r < 4; ++r)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = 16 * r + 4 * lq + e;
      if (i < n) out[(row0 + i) * inner + h * a.vdim + col] = o[r][e] + skip * bf2f(x_s[i * 64 + (((cx >> 3) ^ kv_swz<64>(i)) << 3) + (cx & 7)]);
    }
}

// ---- gate and norms: NTH threads per (token, part); y fp32 [rows][inner].  VEC: four columns per thread and pass
template <typename T, int NTH, bool VEC>
__global__ __launch_bounds__(256) void space_gate_kernel(const T* __restrict__ proj, const float* __restrict__ y, T* __restrict__ out, KvsArgs a) {
  __shared__ float red[4];
  constexpr int W = VEC ? 4 : 1, R = 4;
  const long long t = blockIdx.x;
  const int part = blockIdx.y * (256 / NTH) + threadIdx.x / NTH, lane = threadIdx.x % NTH;
  if (a.tok_kind[t] == 0) return;
  const bool on = part < a.norm_groups;
  const int inner = a.heads * a.vdim, size = inner / a.norm_groups, first = (on ? part : 0) * size;
  const T* zp = proj + t * a.ldp + a.z_off + first;
  const float* yp = y + t * inner + first;
  auto gated = [&](int d) __attribute__((always_inline)) {
    float4 v;
    if constexpr (VEC) {
      v = ld4(yp + d);
      const float4 z = ld4(zp + d);
      v.x *= silu(z.x); v.y *= silu(z.y); v.z *= silu(z.z); v.w *= silu(z.w);
    } else {
      v = make_float4(yp[d] * silu(ld(zp + d)), 0.f, 0.f, 0.f);
    }
    return v;
  };
  float4 kept[R];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int d = (lane + i * NTH) * W;
    kept[i] = d < size ? gated(d) : make_float4(0.f, 0.f, 0.f, 0.f);
    ss += kept[i].x * kept[i].x + kept[i].y * kept[i].y + kept[i].z * kept[i].z + kept[i].w * kept[i].w;
  }
  for (int d = (lane + R * NTH) * W; d < size; d += NTH * W) {
    const float4 v = gated(d);
    ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
  }
  ss = wave_sum(ss);
  if constexpr (NTH == 256) {
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    ss = red[0] + red[1] + red[2] + red[3];
  }
  if (!on) return;
  const float rs = a.out_scale / sqrtf(ss / (float)size + a.eps);
  T* op = out + t * a.ldo + a.o_off + first;
  const float* gp = a.norm + first;
  auto put = [&](int d, float4 v) __attribute__((always_inline)) {
    if constexpr (VEC) {
      const float4 w = ld4(gp + d);
      st4(op + d, make_float4(v.x * rs * w.x, v.y * rs * w.y, v.z * rs * w.z, v.w * rs * w.w));
    } else {
      elem::st(op + d, v.x * rs * gp[d]);
    }
  };
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int d = (lane + i * NTH) * W;
    if (d < size) put(d, kept[i]);
  }
  for (int d = (lane + R * NTH) * W; d < size; d += NTH * W) put(d, gated(d));
}

bool args_ok(const KvsArgs& a) {
  return a.heads > 0 && a.groups > 0 && a.heads % a.groups == 0 && a.dim > 0 && a.dim <= 4096 && a.vdim > 0 && a.vdim <= 1024 && a.dimp == (a.dim + 15) / 16 * 16 && a.dvp == (a.vdim + 15) / 16 * 16 &&
         a.taps > 0 && a.channels == a.heads * a.vdim + 2 * a.groups * a.dim && a.norm_groups > 0 && a.heads * a.vdim % a.norm_groups == 0;
}

template <typename T>
int step(const KvsArgs& a, const void* proj, void* ring, float* y, const int* rows, int n_rows, hipStream_t s) {
  const size_t lds = (size_t)(2 * a.dimp + a.dvp + 256 / (a.dvp / 4) * a.dvp) * 4;
  hipLaunchKernelGGL((space_step_kernel<T>), dim3(n_rows, a.heads), dim3(256), lds, s, (const T*)proj, (T*)ring, y, rows, a);
  return (int)hipGetLastError();
}

template <typename T, int DB, int VB>
int chunk_states(const KvsArgs& a, const T* xbc, float* ws, float* whole, const SpaceChunks& c, int n_chunks, hipStream_t s) {
  constexpr size_t lds = (size_t)CHUNK * (DB + VB + 32) * 4;
  if (lds > 65536 && hipFuncSetAttribute((const void*)space_state_kernel<T, DB, VB>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) return -1;
  const int vb = (a.dvp + VB - 1) / VB;
  hipLaunchKernelGGL((space_state_kernel<T, DB, VB>), dim3(a.heads, n_chunks, (a.dimp + DB - 1) / DB * vb), dim3(256), lds, s, xbc, ws, whole, c, vb, a);
  return (int)hipGetLastError();
}

template <typename T>
int convolve(const KvsArgs& a, const void* proj, const void* ring, T* xbc, float* dts, float* las, int n_rows, hipStream_t s) {
#define KV_SC(VEC, TAPS) \
  hipLaunchKernelGGL((space_conv_kernel<T, VEC, TAPS>), dim3((n_rows + RUN - 1) / RUN, (a.channels + 256 * VEC - 1) / (256 * VEC) + 1), dim3(256), 0, s, (const T*)proj, (const T*)ring, xbc, dts, las, n_rows, a)
  bool done = false;
  if constexpr (sizeof(T) == 2) {
    if (!((a.channels | a.x_off) & 7) && !(a.ldp & 7) && !((uintptr_t)proj & 15)) {
      if (a.taps == 4) KV_SC(8, 4);
      else if (a.taps == 3) KV_SC(8, 3);
      else KV_SC(8, 0);
      done = true;
    }
  }
  if (!done) KV_SC(1, 0);
#undef KV_SC
  return (int)hipGetLastError();
}

template <typename T>
int portions(const KvsArgs& a, const void* proj, void* ring, float* y, void* xbc_, float* f, int n_rows, const int* chunks, int chunk_stride, int n_chunks, const int* segs, int n_segs, const int* first_chunk,
             hipStream_t s) {
  T* xbc = (T*)xbc_;
  float* dts = f;
  float* las = dts + (long long)a.heads * n_rows;
  float* whole = las + (long long)a.heads * n_rows;
  float* ws = whole + ((long long)n_chunks * a.heads + 3) / 4 * 4;
  const SpaceChunks c{chunks, chunks + chunk_stride, n_rows, dts, las};
  int rc = convolve<T>(a, proj, ring, xbc, dts, las, n_rows, s);
  if (rc) return rc;
  const bool d64 = a.dimp <= 64, v64 = a.dvp <= 64, sixteen = sizeof(T) == 2 && !((a.dim | a.vdim | a.channels) & 7) && !((uintptr_t)xbc & 15);
  const int vb = (a.dvp + 63) / 64;
  if constexpr (sizeof(T) == 2) {
    if (sixteen) hipLaunchKernelGGL(space_state16_kernel, dim3(a.heads, n_chunks, (a.dimp + 127) / 128 * vb), dim3(256), 0, s, xbc, ws, whole, c, vb, a);
  }
  if (!sixteen) rc = d64 ? (v64 ? chunk_states<T, 64, 64>(a, xbc, ws, whole, c, n_chunks, s) : chunk_states<T, 64, 128>(a, xbc, ws, whole, c, n_chunks, s))
           : (v64 ? chunk_states<T, 128, 64>(a, xbc, ws, whole, c, n_chunks, s) : chunk_states<T, 128, 128>(a, xbc, ws, whole, c, n_chunks, s));
  if (rc) return rc;
  hipLaunchKernelGGL((space_scan_kernel<T>), dim3((a.dimp * a.dvp / 4 + 255) / 256, a.heads + 1, n_segs), dim3(256), 0, s, (const T*)proj, (T*)ring, ws, whole, segs, segs + n_segs, segs + 2 * n_segs,
                     segs + 3 * n_segs, first_chunk, n_chunks, a);
  if constexpr (sizeof(T) == 2) {
    if (sixteen) {
      hipLaunchKernelGGL(space_out16_kernel, dim3(a.heads, n_chunks, vb), dim3(256), 0, s, xbc, ws, y, c, a);
      return (int)hipGetLastError();
    }
  }
#define KV_SO(NT) hipLaunchKernelGGL((space_out_kernel<T, NT>), dim3(a.heads, n_chunks, (a.dvp + 64 * NT - 1) / (64 * NT)), dim3(256), 0, s, xbc, ws, y, c, a)
  if (a.dvp <= 64) KV_SO(1);
  else KV_SO(2);
#undef KV_SO
  return (int)hipGetLastError();
}

template <typename T>
int gate(const KvsArgs& a, const void* proj, const float* y, void* out, int n_rows, hipStream_t s) {
  const int size = a.heads * a.vdim / a.norm_groups;
  const bool vec = !((size | a.z_off | a.o_off) & 3) && !(a.ldp & 3) && !(a.ldo & 3) && !((uintptr_t)proj & 15) && !((uintptr_t)out & 15);
#define KV_SG(NTH, VEC) \
  hipLaunchKernelGGL((space_gate_kernel<T, NTH, VEC>), dim3(n_rows, (a.norm_groups + 256 / NTH - 1) / (256 / NTH)), dim3(256), 0, s, (const T*)proj, y, (T*)out, a)
  if (size >= 1024) { if (vec) KV_SG(256, true); else KV_SG(256, false); }
  else { if (vec) KV_SG(64, true); else KV_SG(64, false); }
#undef KV_SG
  return (int)hipGetLastError();
}

}  // namespace

extern "C" {

// rows: listed rows that are the only token of their sequence (-1 = unused); y fp32 [rows of the step][heads vdim]
int kvs_step(const KvsArgs* a, const void* proj, void* ring, float* y, int f32, const int* rows, int n_rows, hipStream_t s) {
  if (!args_ok(*a) || n_rows <= 0) return -1;
  return f32 ? step<float>(*a, proj, ring, y, rows, n_rows, s) : step<bf16raw>(*a, proj, ring, y, rows, n_rows, s);
}

// fp32 words of the workspace of kvs_portions
long long kvs_workspace(const KvsArgs* a, int n_rows, int n_chunks) {
  return 2ll * a->heads * n_rows + ((long long)n_chunks * a->heads + 3) / 4 * 4 + (long long)n_chunks * a->heads * a->dimp * a->dvp;
}

// segs: int32 [5][n_segs]: first row, tokens, first position, slot, (unused); portions of at least two tokens are served.
// chunks: int32 [4][chunk_stride]: their pieces of at most 64 tokens (first row, tokens (0 = unused), ...), the first n_chunks in use at most;
// first_chunk [n_segs].  xbc: T [n_rows][channels].
int kvs_portions(const KvsArgs* a, const void* proj, void* ring, float* y, int f32, void* xbc, float* ws, int n_rows, const int* segs, int n_segs, const int* chunks, int chunk_stride, int n_chunks,
                 const int* first_chunk, hipStream_t s) {
  if (!args_ok(*a) || n_segs <= 0 || n_rows <= 0 || n_chunks <= 0 || n_chunks > chunk_stride || n_chunks > 65535 || n_segs > 65535 || ((a->heads * n_rows) & 1)) return -1;
  return f32 ? portions<float>(*a, proj, ring, y, xbc, ws, n_rows, chunks, chunk_stride, n_chunks, segs, n_segs, first_chunk, s)
             : portions<bf16raw>(*a, proj, ring, y, xbc, ws, n_rows, chunks, chunk_stride, n_chunks, segs, n_segs, first_chunk, s);
}

// all rows of the step but padding
int kvs_gate(const KvsArgs* a, const void* proj, const float* y, void* out, int f32, int n_rows, hipStream_t s) {
  if (!args_ok(*a) || n_rows <= 0) return -1;
  return f32 ? gate<float>(*a, proj, y, out, n_rows, s) : gate<bf16raw>(*a, proj, y, out, n_rows, s);
}

}  // extern "C"
