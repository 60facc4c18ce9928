// Retention for gfx950: linear attention with a fixed decay g per head and no softmax.  Per head, with the 32-bit state S [dim, vdim]:
//     S <- g S + k v^T,   o = S^T q,
// q and k rotated (pairs i, i + rot_dims / 2), k times dim^-1/2 behind it.  o leaves divided by its root mean square over vdim and
// multiplied by silu(gate) element by element.  Rotation, scores, state and sums are fp32 (matrix products on the fp32 matrix
// instructions); T is the type of the projections and of the output.
//
//   retention_walk_kernel   token by token: decoding, and portions of value sizes the tile kernels do not take.  A workgroup owns one
//                           head's state, every byte of which is read and written once a token, in whole rows.
//   Portions of several tokens, in chunks of 64 (counted from the portion's start):
//   retention_state_kernel  what a chunk adds to the state, sum_j g^(n-1-j) k_j v_j^T, all chunks and heads at once
//   retention_scan_kernel   the chunks of a portion one after the other, element by element: each chunk's contribution is replaced by the
//                           state in front of it, the last state is kept
//   retention_out_kernel    o_i = g^(i+1) S^T q_i + sum_{j<=i} g^(i-j) (q_i . k_j) v_j, norm and gate, all chunks and heads at once
//
// State: fp32 [slots][heads][dimp][dvp], sizes rounded up to 16 (what is behind dim / vdim stays zero).  A portion that starts at position 0
// takes it as zero, so nothing has to be cleared when a slot changes hands.

#include "elem.h"

struct KvrArgs {
  long long ldp; int q_off, k_off, v_off, g_off;
  const float* log2_decay;                 // [heads]
  const float* cos_t; const float* sin_t;  // [positions][rot_dims / 2]
  int rot_dims, heads, dim, vdim, dimp, dvp;
  float k_scale, eps, out_scale;
  float* state;
  const int* tok_seq; const int* positions; const int* tok_kind;
  long long ldo; int o_off;
};

namespace {
using namespace elem;

constexpr int CHUNK = 64;
typedef __attribute__((ext_vector_type(4))) float f4;

__device__ inline float power(float log2_decay, int n) { return __builtin_amdgcn_exp2f(log2_decay * (float)n); }

// dimension d of a rotated head at position pos (zero behind the head)
template <typename T>
__device__ inline float rotated(const KvrArgs& a, const T* head, int d, int pos) {
  if (d >= a.dim) return 0.f;
  const float x = ld(head + d);
  if (d >= a.rot_dims) return x;
  const int half = a.rot_dims >> 1, i = d < half ? d : d - half;
  const float c = a.cos_t[(long long)pos * half + i], s = a.sin_t[(long long)pos * half + i];
  return d < half ? x * c - ld(head + d + half) * s : x * c + ld(head + d - half) * s;
}
// dimensions d .. d + 3 (d a multiple of four); vec: sizes and offsets are multiples of four, rot_dims of eight
template <typename T>
__device__ inline float4 rotated4(const KvrArgs& a, const T* head, int d, int pos, bool vec) {
  if (!vec) return make_float4(rotated(a, head, d, pos), rotated(a, head, d + 1, pos), rotated(a, head, d + 2, pos), rotated(a, head, d + 3, pos));
  // (no branches: many of these are in flight at a time)
  const bool in = d < a.dim;
  d = in ? d : a.dim - 4;
  float4 x = ld4(head + d);
  if (a.rot_dims) {
    const int half = a.rot_dims >> 1;
    const bool rot = d < a.rot_dims, low = d < half;
    const int i = rot ? (low ? d : d - half) : 0;
    const float4 y = ld4(head + (rot ? (low ? d + half : i) : d)), c = ld4(a.cos_t + (long long)pos * half + i), s = ld4(a.sin_t + (long long)pos * half + i);
    const float f = low ? -1.f : 1.f;
    if (rot) x = make_float4(x.x * c.x + f * y.x * s.x, x.y * c.y + f * y.y * s.y, x.z * c.z + f * y.z * s.z, x.w * c.w + f * y.w * s.w);
  }
  return in ? x : make_float4(0.f, 0.f, 0.f, 0.f);
}
__device__ inline bool vectors(const KvrArgs& a) { return !((a.dim | a.q_off | a.k_off) & 3) && !(a.rot_dims & 7) && !(a.ldp & 3); }

// ---- token by token.  grid (items, heads): listed rows that are the only token of their sequence (rows), or portions of at least min_n
// tokens.  Thread: a group of state rows x 4 columns.
struct WalkItems {
  const int* rows;  // or
  const int* seg_row; const int* seg_n; const int* seg_pos; const int* seg_slot; int min_n;
};

template <typename T>
__global__ __launch_bounds__(256) void retention_walk_kernel(const T* __restrict__ proj, T* __restrict__ out, WalkItems w, KvrArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float part[4];
  const int h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  long long t;
  int n = 1, pos, slot;
  if (w.rows) {
    t = w.rows[blockIdx.x];
    if (t < 0 || a.tok_kind[t] != 1) return;  // unused entry, or a padding row
    pos = a.positions[t];
    slot = a.tok_seq[t];
  } else {
    n = w.seg_n[blockIdx.x];
    if (n < w.min_n || n <= 0) return;
    t = w.seg_row[blockIdx.x];
    pos = w.seg_pos[blockIdx.x];
    slot = w.seg_slot[blockIdx.x];
  }
  const bool vec = vectors(a);
  const float g = power(a.log2_decay[h], 1);
  const int nc = a.dvp >> 2, nrg = 256 / nc;
  const int rg = tid / nc, col = (tid - rg * nc) * 4;
  const bool on = rg < nrg;
  float* qs = sm;               // [dimp]
  float* ks = qs + a.dimp;      // [dimp]
  float* red = ks + a.dimp;     // [nrg][dvp]
  float* st = a.state + ((long long)slot * a.heads + h) * a.dimp * a.dvp + col;
  for (int i = 0; i < n; ++i, ++t, ++pos) {
    const T* pr = proj + t * a.ldp;
    for (int d = tid * 4; d < a.dimp; d += 1024) {
      st4(qs + d, rotated4(a, pr + a.q_off + h * a.dim, d, pos, vec));
      float4 k = rotated4(a, pr + a.k_off + h * a.dim, d, pos, vec);
      k.x *= a.k_scale; k.y *= a.k_scale; k.z *= a.k_scale; k.w *= a.k_scale;
      st4(ks + d, k);
    }
    float v[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = on && col + e < a.vdim ? ld(pr + a.v_off + h * a.vdim + col + e) : 0.f;
    constexpr int U = 8;
    float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
    float4 s[U];
    auto fetch = [&](int r0) __attribute__((always_inline)) {
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int r = r0 + u * nrg;
        s[u] = on && r < a.dimp && pos > 0 ? ld4(st + (long long)r * a.dvp) : make_float4(0.f, 0.f, 0.f, 0.f);
      }
    };
    fetch(rg);
    __syncthreads();
    for (int r0 = rg; r0 < a.dimp; r0 += U * nrg) {
      if (r0 != rg) fetch(r0);
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int r = r0 + u * nrg;
        if (on && r < a.dimp) {
          const float k = ks[r], q = qs[r];
          s[u].x = s[u].x * g + k * v[0]; s[u].y = s[u].y * g + k * v[1]; s[u].z = s[u].z * g + k * v[2]; s[u].w = s[u].w * g + k * v[3];
          o.x += q * s[u].x; o.y += q * s[u].y; o.z += q * s[u].z; o.w += q * s[u].w;
          st4(st + (long long)r * a.dvp, s[u]);
        }
      }
    }
    if (on) st4(red + rg * a.dvp + col, o);
    __syncthreads();
    float ss = 0.f;
    for (int d = tid; d < a.vdim; d += 256) {
      float x = 0.f;
      for (int r = 0; r < nrg; ++r) x += red[r * a.dvp + d];
      red[d] = x;  // (row group 0's partial of this column, read by this thread only)
      ss += x * x;
    }
    ss = wave_sum(ss);
    if (lane == 0) part[wave] = ss;
    __syncthreads();
    const float rs = a.out_scale / sqrtf((part[0] + part[1] + part[2] + part[3]) / (float)a.vdim + a.eps);
    for (int d = tid; d < a.vdim; d += 256) elem::st(out + t * a.ldo + a.o_off + h * a.vdim + d, red[d] * rs * silu(ld(pr + a.g_off + h * a.vdim + d)));
    if (i + 1 < n) __syncthreads();  // (the next token reuses the LDS; its state rows are this thread's own)
  }
}

// ---- a chunk's contribution to the state: grid (heads, chunks, blocks of DB x VB); 4 waves, a quarter of the block each
struct Chunks { const int* row; const int* n; const int* pos; };

template <typename T, int DB, int VB>
__global__ __launch_bounds__(256) void retention_state_kernel(const T* __restrict__ proj, float* __restrict__ ws, Chunks c, int v_blocks, KvrArgs a) {
  constexpr int KS = DB + 16, VS = VB + 16;  // (a fragment's four rows lie in different banks)
  constexpr int ND = DB / 32, NV = VB / 32;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* k_s = sm;             // [CHUNK][KS]
  float* v_s = sm + CHUNK * KS;  // [CHUNK][VS]
  const int h = blockIdx.x, b = blockIdx.y;
  const int n = c.n[b];
  if (n <= 0) return;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, lr = lane & 15, lq = lane >> 4;
  const int d_blk = blockIdx.z / v_blocks * DB, v_blk = blockIdx.z % v_blocks * VB;
  const long long row0 = c.row[b];
  const int pos0 = c.pos[b];
  const bool vec = vectors(a), v_vec = !((a.vdim | a.v_off) & 3) && !(a.ldp & 3);
  const float lg = a.log2_decay[h];
  const int rows = (n + 3) & ~3;
#pragma unroll 4
  for (int i = tid; i < rows * (DB / 4); i += 256) {
    const int j = i / (DB / 4), d = i % (DB / 4) * 4;
    const int jr = j < n ? j : n - 1;
    float4 k = rotated4(a, proj + (row0 + jr) * a.ldp + a.k_off + h * a.dim, d_blk + d, pos0 + jr, vec);
    const float f = j < n ? a.k_scale * power(lg, n - 1 - j) : 0.f;
    k.x *= f; k.y *= f; k.z *= f; k.w *= f;
    st4(k_s + j * KS + d, k);
  }
#pragma unroll 4
  for (int i = tid; i < rows * (VB / 4); i += 256) {
    const int j = i / (VB / 4), d = i % (VB / 4) * 4, vd = v_blk + d;
    const T* p = proj + (row0 + (j < n ? j : n - 1)) * a.ldp + a.v_off + h * a.vdim;  // (keys past the last one are zero)
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    if (v_vec) {
      v = ld4(p + (vd < a.vdim ? vd : a.vdim - 4));
      if (vd >= a.vdim) v = make_float4(0.f, 0.f, 0.f, 0.f);
    } else {
      if (vd < a.vdim) v.x = ld(p + vd);
      if (vd + 1 < a.vdim) v.y = ld(p + vd + 1);
      if (vd + 2 < a.vdim) v.z = ld(p + vd + 2);
      if (vd + 3 < a.vdim) v.w = ld(p + vd + 3);
    }
    st4(v_s + j * VS + d, v);
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

// ---- portions: grid (elements / 1024, heads, portions), four elements per thread
__global__ __launch_bounds__(256) void retention_scan_kernel(float* __restrict__ ws, const int* __restrict__ seg_n, const int* __restrict__ seg_pos, const int* __restrict__ seg_slot,
                                                             const int* __restrict__ first_chunk, int n_chunks, KvrArgs a) {
  const int h = blockIdx.y, sg = blockIdx.z;
  const int n = seg_n[sg];
  if (n < 2) return;
  const int size = a.dimp * a.dvp, i = (blockIdx.x * 256 + threadIdx.x) * 4;
  const int c0 = first_chunk[sg], nc = (n + CHUNK - 1) / CHUNK;
  if (i >= size || c0 < 0 || c0 + nc > n_chunks) return;
  float* st = a.state + ((long long)seg_slot[sg] * a.heads + h) * size + i;
  float* u = ws + ((long long)c0 * a.heads + h) * size + i;
  const long long step = (long long)a.heads * size;
  const float lg = a.log2_decay[h], whole = power(lg, CHUNK);
  float4 s = seg_pos[sg] > 0 ? ld4(st) : make_float4(0.f, 0.f, 0.f, 0.f);
  constexpr int U = 4;  // chunks in flight
  for (int c = 0; c < nc; c += U) {
    float4 x[U];
#pragma unroll
    for (int e = 0; e < U; ++e) x[e] = c + e < nc ? ld4(u + (c + e) * step) : make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int e = 0; e < U; ++e) {
      if (c + e >= nc) break;
      st4(u + (c + e) * step, s);
      const float f = c + e + 1 < nc ? whole : power(lg, n - (nc - 1) * CHUNK);
      s.x = s.x * f + x[e].x; s.y = s.y * f + x[e].y; s.z = s.z * f + x[e].z; s.w = s.w * f + x[e].w;
    }
  }
  st4(st, s);
}

// ---- outputs: grid (heads, chunks).  The waves share the columns of o (NT tiles of 16 each), so the state and the values are read once per
// workgroup, straight from memory; queries and keys pass through LDS in blocks of 64 dimensions.
template <typename T, int NT>
__global__ __launch_bounds__(256, NT <= 2 ? 3 : 2) void retention_out_kernel(const T* __restrict__ proj, const float* __restrict__ ws, T* __restrict__ out, Chunks c, KvrArgs a) {
  constexpr int S = CHUNK + 4;  // (16 rows x 4 entries of a fragment lie in different banks)
  __shared__ __attribute__((aligned(16))) float q_s[CHUNK * S], k_s[CHUNK * S], p_s[CHUNK * S];
  __shared__ float sums[4][CHUNK];
  const int h = blockIdx.x, b = blockIdx.y;
  const int n = c.n[b];
  if (n <= 0) return;
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, lr = lane & 15, lq = lane >> 4;
  const long long row0 = c.row[b];
  const int pos0 = c.pos[b];
  const bool vec = vectors(a);
  const float lg = a.log2_decay[h];
  const int tiles = a.dvp / 16;
  const float* s_in = ws + ((long long)b * a.heads + h) * a.dimp * a.dvp;
  const int rts = (n + 15) >> 4;  // row tiles in use
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
    col[y] = 16 * (wave * NT + y < tiles ? wave * NT + y : tiles - 1) + lr;
    vcol[y] = col[y] < a.vdim ? col[y] : a.vdim - 1;
    live[y] = wave * NT + y < tiles && col[y] < a.vdim;
  }
  for (int db = 0; db < a.dimp; db += 64) {
    if (db) __syncthreads();
    const int nd = a.dimp - db < 64 ? a.dimp - db : 64;  // (a multiple of 16)
    float sb[16][NT];  // the block's rows of the state: on their way while queries and keys are rotated
#pragma unroll
    for (int u = 0; u < 16; ++u)
#pragma unroll
      for (int y = 0; y < NT; ++y) sb[u][y] = s_in[(long long)(4 * u < nd ? db + 4 * u + lq : lq) * a.dvp + col[y]];
#pragma unroll 4
    for (int i = tid; i < CHUNK * 16; i += 256) {
      const int j = i >> 4, d = (i & 15) * 4;
      const int jr = j < n ? j : n - 1;  // (rows past the last one: it again, never used)
      const T* pr = proj + (row0 + jr) * a.ldp + h * a.dim;
      const float4 q = rotated4(a, pr + a.q_off, db + d, pos0 + jr, vec);
      float4 k = rotated4(a, pr + a.k_off, db + d, pos0 + jr, vec);
      k.x *= a.k_scale; k.y *= a.k_scale; k.z *= a.k_scale; k.w *= a.k_scale;
      st4(q_s + j * S + d, q);
      st4(k_s + j * S + d, k);
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
  float vb[16][NT];  // the values: on their way while the scores are weighted
#pragma unroll
  for (int u = 0; u < 16; ++u) {
    const int j = 4 * u + lq;
    const T* vp = proj + (row0 + (j < n ? j : n - 1)) * a.ldp + a.v_off + h * a.vdim;  // (rows past the last one have weight zero)
#pragma unroll
    for (int y = 0; y < NT; ++y) vb[u][y] = ld(vp + vcol[y]);
  }
  // scores of row tile `wave`, weighted; o so far, decayed
#pragma unroll
  for (int x = 0; x < 4; ++x)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = 16 * wave + 4 * lq + e, j = 16 * x + lr;
      p_s[i * S + j] = j <= i && i < n ? p[x][e] * power(lg, i - j) : 0.f;
    }
#pragma unroll
  for (int r = 0; r < 4; ++r)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float f = power(lg, 16 * r + 4 * lq + e + 1);
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
  float gz[16][NT];  // the gates
#pragma unroll
  for (int u = 0; u < 16; ++u) {
    const int i = 16 * (u >> 2) + 4 * lq + (u & 3);
    const T* gp = proj + (row0 + (i < n ? i : n - 1)) * a.ldp + a.g_off + h * a.vdim;
#pragma unroll
    for (int y = 0; y < NT; ++y) gz[u][y] = ld(gp + vcol[y]);
  }
#pragma unroll
  for (int u = 0; u < 16; ++u) {
    float ss = 0.f;
#pragma unroll
    for (int y = 0; y < NT; ++y) ss += live[y] ? o[u >> 2][y][u & 3] * o[u >> 2][y][u & 3] : 0.f;
#pragma unroll
    for (int m = 1; m < 16; m <<= 1) ss += __shfl_xor(ss, m, 64);
    if (lr == 0) sums[wave][16 * (u >> 2) + 4 * lq + (u & 3)] = ss;
  }
  __syncthreads();
#pragma unroll
  for (int u = 0; u < 16; ++u) {
    const int i = 16 * (u >> 2) + 4 * lq + (u & 3);
    const float rs = a.out_scale / sqrtf((sums[0][i] + sums[1][i] + sums[2][i] + sums[3][i]) / (float)a.vdim + a.eps);
    T* op = out + (row0 + i) * a.ldo + a.o_off + h * a.vdim;
#pragma unroll
    for (int y = 0; y < NT; ++y)
      if (i < n && live[y]) st(op + col[y], o[u >> 2][y][u & 3] * rs * silu(gz[u][y]));
  }
}

bool args_ok(const KvrArgs& a) {
  return a.heads > 0 && a.dim > 0 && a.dim <= 1024 && a.vdim > 0 && a.vdim <= 1024 && a.dimp == (a.dim + 15) / 16 * 16 && a.dvp == (a.vdim + 15) / 16 * 16 && a.rot_dims >= 0 && a.rot_dims <= a.dim &&
         !(a.rot_dims & 1);
}

template <typename T>
int walk(const KvrArgs& a, const void* proj, void* out, const WalkItems& w, int items, hipStream_t s) {
  const size_t lds = (size_t)(2 * a.dimp + 256 / (a.dvp / 4) * a.dvp) * 4;
  hipLaunchKernelGGL((retention_walk_kernel<T>), dim3(items, a.heads), dim3(256), lds, s, (const T*)proj, (T*)out, w, a);
  return (int)hipGetLastError();
}

template <typename T, int DB, int VB>
int chunk_states(const KvrArgs& a, const void* proj, float* ws, const Chunks& c, int n_chunks, hipStream_t s) {
  constexpr size_t lds = (size_t)CHUNK * (DB + VB + 32) * 4;
  if (lds > 65536 && hipFuncSetAttribute((const void*)retention_state_kernel<T, DB, VB>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) return -1;
  const int vb = (a.dvp + VB - 1) / VB;
  hipLaunchKernelGGL((retention_state_kernel<T, DB, VB>), dim3(a.heads, n_chunks, (a.dimp + DB - 1) / DB * vb), dim3(256), lds, s, (const T*)proj, ws, c, vb, a);
  return (int)hipGetLastError();
}

template <typename T>
int portions(const KvrArgs& a, const void* proj, void* out, float* ws, const Chunks& c, int n_chunks, const int* segs, int n_segs, const int* first_chunk, hipStream_t s) {
  const bool d64 = a.dimp <= 64, v64 = a.dvp <= 64;
  int rc = d64 ? (v64 ? chunk_states<T, 64, 64>(a, proj, ws, c, n_chunks, s) : chunk_states<T, 64, 128>(a, proj, ws, c, n_chunks, s))
               : (v64 ? chunk_states<T, 128, 64>(a, proj, ws, c, n_chunks, s) : chunk_states<T, 128, 128>(a, proj, ws, c, n_chunks, s));
  if (rc) return rc;
  hipLaunchKernelGGL(retention_scan_kernel, dim3((a.dimp * a.dvp / 4 + 255) / 256, a.heads, n_segs), dim3(256), 0, s, ws, segs + n_segs, segs + 2 * n_segs, segs + 3 * n_segs, first_chunk, n_chunks, a);
  const dim3 grid(a.heads, n_chunks);
#define KV_RO(NT) hipLaunchKernelGGL((retention_out_kernel<T, NT>), grid, dim3(256), 0, s, (const T*)proj, ws, (T*)out, c, a)
  if (a.dvp <= 64) KV_RO(1);
  else if (a.dvp <= 128) KV_RO(2);
  else KV_RO(4);
#undef KV_RO
  return (int)hipGetLastError();
}

}  // namespace

extern "C" {

// value sizes the chunk kernels take
int kvr_chunked(int vdim) { return vdim <= 256; }

// rows: listed rows that are the only token of their sequence (-1 = unused)
int kvr_rows(const KvrArgs* a, const void* proj, void* out, int f32, const int* rows, int n_rows, hipStream_t s) {
  if (!args_ok(*a) || n_rows <= 0) return -1;
  const WalkItems w{rows, nullptr, nullptr, nullptr, nullptr, 0};
  return f32 ? walk<float>(*a, proj, out, w, n_rows, s) : walk<bf16raw>(*a, proj, out, w, n_rows, s);
}

// segs: int32 [5][n_segs]: first row, tokens, first position, slot, (unused); portions of at least two tokens are served.
// chunks: int32 [4][chunk_stride]: their pieces of at most 64 tokens (tokens 0 = unused), the first n_chunks in use at most; first_chunk
// [n_segs].  ws: fp32 [n_chunks][heads][dimp][dvp].  n_chunks 0: token by token.
int kvr_portions(const KvrArgs* a, const void* proj, void* out, int f32, const int* segs, int n_segs, const int* chunks, int chunk_stride, int n_chunks, const int* first_chunk, float* ws, hipStream_t s) {
  if (!args_ok(*a) || n_segs <= 0) return -1;
  if (n_chunks == 0) {
    const WalkItems w{nullptr, segs, segs + n_segs, segs + 2 * n_segs, segs + 3 * n_segs, 2};
    return f32 ? walk<float>(*a, proj, out, w, n_segs, s) : walk<bf16raw>(*a, proj, out, w, n_segs, s);
  }
  if (n_chunks < 0 || n_chunks > chunk_stride || !kvr_chunked(a->vdim) || !ws) return -1;
  const Chunks c{chunks, chunks + chunk_stride, chunks + 2 * chunk_stride};
  return f32 ? portions<float>(*a, proj, out, ws, c, n_chunks, segs, n_segs, first_chunk, s) : portions<bf16raw>(*a, proj, out, ws, c, n_chunks, segs, n_segs, first_chunk, s);
}

}  // extern "C"
