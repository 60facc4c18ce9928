// Mixture of experts for gfx950: routing, the grouping of (token, choice) pairs by expert, and the experts' products for few rows (the
// products for many rows are the tiled GEMM's grouped form, csrc/wide_gemm.hip).
//
// A pair p = token * top + choice; expert_of[p] is its expert (-1: the row is padding and chooses nobody), weight_of[p] its weight.  Matrices
// of all experts are stacked; in bf16 in MFMA fragment order [N / 16][K / 32][64][8], an expert's first tile at expert * N / 16.  Gate and up
// rows are interleaved in eights.

#include "attn_tiles.h"
#include "experts.h"

namespace {
using namespace elem;
using namespace attn;

// ---- routing: logits (fp32 products, plus a bias), scores sigmoid(logit), softmax(logits), or softmax over the chosen logits alone (the
// scores to choose by are then the logits), the `top` largest score + correction (the first of equals), their scores times `scale`.  With shared_of, row E of the router is the shared expert's gate: its sigmoid.
// Workgroup: 16 tokens, 16 waves — which share K (bf16, matrix cores) or take a token each (fp32), then choose for a token each.
enum Scores { SIGMOID = 0, SOFTMAX = 1, CHOSEN = 2 };
struct RouteArgs {
  int T, E, Ep, top, K; long long ldh;  // Ep: experts in the packed matrix (a multiple of 16)
  const float* correction; const int* slots;
  int* expert_of; float* weight_of;
  int scores; float scale; float* shared_of;  // scores: a Scores
  const float* bias;
};

// NC: experts per lane of a token's wave; TL: tiles of 16 experts multiplied at a time (bf16)
template <typename T, int NC, int TL>
__global__ __launch_bounds__(1024) void route_kernel(const T* __restrict__ h, const T* __restrict__ w, RouteArgs a) {
  extern __shared__ __attribute__((aligned(16))) float rt_lds[];  // logits [16][Ep + 1], then (bf16) partial sums [16 waves][16 TL][16]
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, lr = lane & 15, lq = lane >> 4;
  const int t0 = blockIdx.x * 16, ls = a.Ep + 1;
  if constexpr (sizeof(T) == 2) {
    float* part = rt_lds + (16 * ls + 3) / 4 * 4;
    constexpr int U = 4;
    const int nks = a.K / 32, k0 = nks * wave / 16, k1 = nks * (wave + 1) / 16;
    const int t = t0 + lr < a.T ? t0 + lr : a.T - 1;
    const T* hp = h + (long long)t * a.ldh + lq * 8;
    for (int e0 = 0; e0 < a.Ep; e0 += 16 * TL) {
      const int nt = a.Ep - e0 >= 16 * TL ? TL : (a.Ep - e0) / 16;
      const frag_ab* wp = reinterpret_cast<const frag_ab*>(w) + (long long)(e0 / 16) * nks * 64 + lane;
      frag_acc4 acc[TL];
#pragma unroll
      for (int i = 0; i < TL; ++i) acc[i] = (frag_acc4){0.f, 0.f, 0.f, 0.f};
      for (int ks = k0; ks < k1; ks += U) {
        frag_ab x[U], m[U][TL];
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int k = ks + u < k1 ? ks + u : k1 - 1;  // (steps past the end are not multiplied)
          x[u] = *reinterpret_cast<const frag_ab*>(hp + k * 32);
#pragma unroll
          for (int i = 0; i < TL; ++i) m[u][i] = wp[((long long)(i < nt ? i : nt - 1) * nks + k) * 64];
        }
#pragma unroll
        for (int u = 0; u < U; ++u)
          if (ks + u < k1) {
#pragma unroll
            for (int i = 0; i < TL; ++i) acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(m[u][i], x[u], acc[i], 0, 0, 0);
          }
      }
#pragma unroll
      for (int i = 0; i < TL; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) part[(wave * 16 * TL + 16 * i + 4 * lq + e) * 16 + lr] = acc[i][e];
      __syncthreads();
      for (int i = tid; i < nt * 256; i += 1024) {
        float s = 0.f;
#pragma unroll
        for (int k = 0; k < 16; ++k) s += part[k * 256 * TL + i];
        const int e = e0 + (i >> 4);
        rt_lds[(i & 15) * ls + e] = a.bias && e < a.E ? s + a.bias[e] : s;
      }
      __syncthreads();
    }
  } else {
    const int t = t0 + wave < a.T ? t0 + wave : a.T - 1;
    const T* hp = h + (long long)t * a.ldh;
    for (int e = 0; e < a.E + (a.shared_of ? 1 : 0); ++e) {
      float s = 0.f;
      for (int k = lane; k < a.K; k += 64) s += ld(hp + k) * ld(w + (long long)e * a.K + k);
      s = wave_sum(s);
      if (lane == 0) rt_lds[wave * ls + e] = a.bias && e < a.E ? s + a.bias[e] : s;
    }
    __syncthreads();
  }
  const int t = t0 + wave;
  if (t >= a.T) return;
  const bool pad = a.slots[t] < 0;
  const float* z = rt_lds + wave * ls;
  if (a.shared_of && lane == 0) a.shared_of[t] = pad ? 0.f : 1.f / (1.f + expf(-z[a.E]));
  float top_z = 0.f, unit = 1.f;  // a score: sigmoid(z), or exp(z - top_z) over the sum of them
  if (a.scores != SIGMOID) {
    top_z = -INFINITY;
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < NC; ++i)
      if (lane + 64 * i < a.E) top_z = fmaxf(top_z, z[lane + 64 * i]);
    top_z = wave_max(top_z);
#pragma unroll
    for (int i = 0; i < NC; ++i)
      if (lane + 64 * i < a.E) sum += expf(z[lane + 64 * i] - top_z);
    unit = 1.f / wave_sum(sum);
  }
  auto score = [&](int e) { return a.scores != SIGMOID ? expf(z[e] - top_z) * unit : 1.f / (1.f + expf(-z[e])); };
  float c[NC];
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int e = lane + 64 * i;
    c[i] = e < a.E ? (a.scores == CHOSEN ? z[e] : score(e)) + a.correction[e] : -INFINITY;
    if (!(c[i] == c[i])) c[i] = -INFINITY;  // (padding rows may hold anything: every choice below must be written all the same)
  }
  if constexpr (NC == 1) {  // an expert per lane: its rank is the number of better ones (of equals, the earlier)
    int rank = 0;
#pragma unroll
    for (int j = 0; j < 64; ++j) {
      const float o = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(c[0]), j));
      rank += (o > c[0] || (o == c[0] && j < lane)) ? 1 : 0;
    }
    if (a.scores == CHOSEN) unit = 1.f / wave_sum(lane < a.E && rank < a.top ? expf(z[lane] - top_z) : 0.f);
    if (lane < a.E && rank < a.top) {
      a.expert_of[t * a.top + rank] = pad ? -1 : lane;
      a.weight_of[t * a.top + rank] = pad ? 0.f : score(lane) * a.scale;
    }
    return;
  }
  int mine = -1;  // lane k: choice k
  for (int k = 0; k < a.top; ++k) {
    float best = -INFINITY;
    int idx = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < NC; ++i)
      if (c[i] > best) { best = c[i]; idx = lane + 64 * i; }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float v = __shfl_xor(best, o, 64);
      const int j = __shfl_xor(idx, o, 64);
      if (v > best || (v == best && j < idx)) { best = v; idx = j; }
    }
    if (lane == k) mine = idx;
#pragma unroll
    for (int i = 0; i < NC; ++i)
      if (lane + 64 * i == idx) c[i] = -INFINITY;
  }
  const bool ok = !pad && lane < a.top && mine >= 0 && mine < a.E;
  if (a.scores == CHOSEN) unit = 1.f / wave_sum(ok ? expf(z[mine] - top_z) : 0.f);
  if (lane >= a.top) return;
  a.expert_of[t * a.top + lane] = ok ? mine : -1;
  a.weight_of[t * a.top + lane] = ok ? score(mine) * a.scale : 0.f;
}

// ---- grouping for many rows: pairs in the order of their experts, cut into tiles of at most `bm` pairs.  One workgroup.
__global__ __launch_bounds__(1024) void group_pairs_kernel(const int* __restrict__ expert_of, int n_pairs, int E, int bm, GroupedRows g) {
  __shared__ int cnt[1024], off[1024], tiles[1024];
  const int e = threadIdx.x;
  cnt[e] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < n_pairs; i += 1024) {
    const int x = expert_of[i];
    if (x >= 0) atomicAdd(&cnt[x], 1);
  }
  __syncthreads();
  const int mine = cnt[e], my_tiles = (mine + bm - 1) / bm;
  off[e] = mine;
  tiles[e] = my_tiles;
  __syncthreads();
  for (int d = 1; d < 1024; d <<= 1) {  // running sums
    const int a = e >= d ? off[e - d] : 0, b = e >= d ? tiles[e - d] : 0;
    __syncthreads();
    off[e] += a;
    tiles[e] += b;
    __syncthreads();
  }
  const int first = off[e] - mine, tile0 = tiles[e] - my_tiles;
  for (int i = 0; i < my_tiles; ++i) {
    if (tile0 + i >= g.max_tiles) break;
    g.tile_expert[tile0 + i] = e;
    g.tile_first[tile0 + i] = first + i * bm;
    g.tile_rows[tile0 + i] = mine - i * bm < bm ? mine - i * bm : bm;
  }
  if (e == 1023) g.n_tiles[0] = tiles[e] < g.max_tiles ? tiles[e] : g.max_tiles;
  cnt[e] = first;
  __syncthreads();
  for (int i = threadIdx.x; i < n_pairs; i += 1024) {
    const int x = expert_of[i];
    if (x >= 0) g.order[atomicAdd(&cnt[x], 1)] = i;
  }
}

// ---- products for few rows (at most 128 tokens): workgroup = 32 features of one expert; its four waves share K and stream the weights once
// for up to 64 of the expert's rows.  Rows of x: pair / row_div.  MODE GATED: y[pair][N / 2] = gate(gate, up); SQUARED: y[pair][N] = max(., 0)^2;
// PLAIN: y[pair][N].
struct ExpertRowsArgs {
  const int* expert_of; int n_pairs, row_div;
  int N, K; long long ldx, ldy;
  ExpertGate gate;
};

enum RowsMode { PLAIN = 0, GATED = 1, SQUARED = 2 };
__device__ inline float relu2(float v) { v = fmaxf(v, 0.f); return v * v; }

template <int NT, int MODE>
__device__ inline void expert_rows(const frag_ab* __restrict__ w, const bf16raw* __restrict__ x, bf16raw* __restrict__ y, const ExpertRowsArgs& a, const int* list, int n, int n0, float* red) {
  constexpr int NF = 2, U = 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, lr = lane & 15, lq = lane >> 4;
  const int nks = a.K / 32, mine = (nks - wave + 3) / 4;  // k-steps wave, wave + 4, ...
  const bf16raw* xp[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j) {
    const int r = 16 * j + lr;
    xp[j] = x + (long long)(list[r < n ? r : n - 1] / a.row_div) * a.ldx + lq * 8;
  }
  frag_acc4 acc[NF][NT];
#pragma unroll
  for (int f = 0; f < NF; ++f)
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[f][j] = (frag_acc4){0.f, 0.f, 0.f, 0.f};
  frag_ab wa[2][U][NF], xa[2][U][NT];
  auto fetch = [&](int set, int g) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      int i = g * U + u;
      i = i < mine ? i : mine - 1;  // (steps past the end are not multiplied)
      const int ks = wave + 4 * i;
#pragma unroll
      for (int f = 0; f < NF; ++f) wa[set][u][f] = __builtin_nontemporal_load(w + ((long long)f * nks + ks) * 64 + lane);
#pragma unroll
      for (int j = 0; j < NT; ++j) xa[set][u][j] = *reinterpret_cast<const frag_ab*>(xp[j] + ks * 32);
    }
  };
  auto multiply = [&](int set, int g) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (g * U + u < mine) {
#pragma unroll
        for (int f = 0; f < NF; ++f)
#pragma unroll
          for (int j = 0; j < NT; ++j) acc[f][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wa[set][u][f], xa[set][u][j], acc[f][j], 0, 0, 0);
      }
  };
  if (mine > 0) {
    const int groups = (mine + U - 1) / U;
    fetch(0, 0);
    for (int g = 0; g < groups; g += 2) {
      if (g + 1 < groups) fetch(1, g + 1);
      multiply(0, g);
      if (g + 1 < groups) {
        if (g + 2 < groups) fetch(0, g + 2);
        multiply(1, g + 1);
      }
    }
  }
#pragma unroll
  for (int f = 0; f < NF; ++f)
#pragma unroll
    for (int j = 0; j < NT; ++j) st4(red + ((wave * NF + f) * NT + j) * 256 + lane * 4, make_float4(acc[f][j][0], acc[f][j][1], acc[f][j][2], acc[f][j][3]));
  __syncthreads();
  for (int i = wave; i < NF * NT; i += 4) {
    const int f = i / NT, j = i % NT;
    float4 v = ld4(red + i * 256 + lane * 4);
#pragma unroll
    for (int k = 1; k < 4; ++k) {
      const float4 b = ld4(red + (k * NF * NT + i) * 256 + lane * 4);
      v.x += b.x; v.y += b.y; v.z += b.z; v.w += b.w;
    }
    const int r = 16 * j + lr;
    const long long pair = list[r < n ? r : n - 1];
    if constexpr (MODE == GATED) {  // lanes of the upper half hold the up rows of the lower half's features
      float4 u;
      u.x = __shfl_xor(v.x, 32, 64); u.y = __shfl_xor(v.y, 32, 64); u.z = __shfl_xor(v.z, 32, 64); u.w = __shfl_xor(v.w, 32, 64);
      if (lq < 2 && r < n)
        st4(y + pair * a.ldy + n0 / 2 + 8 * f + 4 * lq, make_float4(expert_gate(v.x, u.x, a.gate), expert_gate(v.y, u.y, a.gate), expert_gate(v.z, u.z, a.gate), expert_gate(v.w, u.w, a.gate)));
    } else if (r < n) {
      if constexpr (MODE == SQUARED) v = make_float4(relu2(v.x), relu2(v.y), relu2(v.z), relu2(v.w));
      st4(y + pair * a.ldy + n0 + 16 * f + 4 * lq, v);
    }
  }
  __syncthreads();
}

template <int MODE>
__global__ __launch_bounds__(256) void expert_rows_kernel(const bf16raw* __restrict__ w, const bf16raw* __restrict__ x, bf16raw* __restrict__ y, ExpertRowsArgs a) {
  __shared__ int list[128];
  __shared__ int counts[4];
  __shared__ __attribute__((aligned(16))) float red[4 * 2 * 4 * 256];
  const int e = blockIdx.y, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  // the expert's pairs, in order: every wave looks through a quarter of them
  const int per = (a.n_pairs + 255) / 256 * 64, lo = wave * per, hi = lo + per < a.n_pairs ? lo + per : a.n_pairs;
  int c = 0;
  for (int i = lo; i < hi; i += 64) c += __builtin_popcountll(__builtin_amdgcn_ballot_w64(i + lane < hi && a.expert_of[i + lane] == e));
  if (lane == 0) counts[wave] = c;
  __syncthreads();
  int at = 0, n = 0;
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    if (k < wave) at += counts[k];
    n += counts[k];
  }
  if (n == 0) return;
  for (int i = lo; i < hi; i += 64) {
    const bool hit = i + lane < hi && a.expert_of[i + lane] == e;
    const unsigned long long m = __builtin_amdgcn_ballot_w64(hit);
    const int p = at + __builtin_popcountll(m & ((1ull << lane) - 1));
    if (hit && p < 128) list[p] = i + lane;
    at += __builtin_popcountll(m);
  }
  n = n < 128 ? n : 128;  // (a token chooses an expert once: at most as many as tokens)
  __syncthreads();
  const int n0 = blockIdx.x * 32;
  const frag_ab* wp = reinterpret_cast<const frag_ab*>(w) + (long long)(e * a.N + n0) / 16 * (a.K / 32) * 64;
  for (int r = 0; r < n; r += 64) {
    const int left = n - r;
    if (left <= 16) expert_rows<1, MODE>(wp, x, y, a, list + r, left, n0, red);
    else if (left <= 32) expert_rows<2, MODE>(wp, x, y, a, list + r, left, n0, red);
    else expert_rows<4, MODE>(wp, x, y, a, list + r, left < 64 ? left : 64, n0, red);
  }
}

// ---- fp32: one workgroup per pair, one wave per feature at a time
template <int MODE>
__global__ __launch_bounds__(256) void expert_pairs_kernel(const float* __restrict__ w, const float* __restrict__ x, float* __restrict__ y, ExpertRowsArgs a) {
  const int p = blockIdx.x, e = a.expert_of[p], wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  if (e < 0) return;
  const float* xr = x + (long long)(p / a.row_div) * a.ldx;
  const float* we = w + (long long)e * a.N * a.K;
  for (int n = wave; n < (MODE == GATED ? a.N / 2 : a.N); n += 4) {
    const float* w0 = we + (long long)(MODE == GATED ? n / 8 * 16 + n % 8 : n) * a.K;
    float s = 0.f, u = 0.f;
    for (int k = lane * 4; k < a.K; k += 256) {
      const float4 xv = ld4(xr + k), wv = ld4(w0 + k);
      s += xv.x * wv.x + xv.y * wv.y + xv.z * wv.z + xv.w * wv.w;
      if constexpr (MODE == GATED) {
        const float4 uv = ld4(w0 + (long long)8 * a.K + k);
        u += xv.x * uv.x + xv.y * uv.y + xv.z * uv.z + xv.w * uv.w;
      }
    }
    s = wave_sum(s);
    if constexpr (MODE == GATED) { u = wave_sum(u); s = expert_gate(s, u, a.gate); }
    if constexpr (MODE == SQUARED) s = relu2(s);
    if (lane == 0) y[(long long)p * a.ldy + n] = s;
  }
}

}  // namespace

extern "C" {

int kve_route(const void* h, int f32, long long ldh, const void* w, const float* correction, const int* slots, int T, int E, int Ep, int top, int K, int* expert_of, float* weight_of, int scores, float scale, float* shared_of, const float* bias,
              hipStream_t s) {
  if (T <= 0 || E <= 0 || E > 1024 || Ep < E + (shared_of ? 1 : 0) || top <= 0 || top > E || top > 64 || K <= 0 || scores < SIGMOID || scores > CHOSEN || (!f32 && ((Ep & 15) || (K & 31) || (ldh & 7)))) return -1;
  const RouteArgs a{T, E, Ep, top, K, ldh, correction, slots, expert_of, weight_of, scores, scale, shared_of, bias};
  const int tl = Ep > 64 && Ep <= 80 ? 5 : 4;  // (64 experts and a shared one: all at a time)
  const size_t lds = ((size_t)16 * (Ep + 1) + 4 + (f32 ? 0 : 16 * 16 * tl * 16)) * 4;
  const dim3 grid((T + 15) / 16);
#define KV_RT(Tt, NC, TL)                                                                                                                                                 \
  do {                                                                                                                                                                    \
    if (lds > 65536 && hipFuncSetAttribute((const void*)route_kernel<Tt, NC, TL>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) return -1;          \
    hipLaunchKernelGGL((route_kernel<Tt, NC, TL>), grid, dim3(1024), lds, s, (const Tt*)h, (const Tt*)w, a);                                                               \
  } while (0)
#define KV_RTL(Tt, NC) do { if (tl == 5) KV_RT(Tt, NC, 5); else KV_RT(Tt, NC, 4); } while (0)
#define KV_RT2(Tt) do { if (E <= 64) KV_RTL(Tt, 1); else if (E <= 256) KV_RTL(Tt, 4); else KV_RT(Tt, 16, 4); } while (0)
  if (f32) KV_RT2(float);
  else KV_RT2(bf16raw);
#undef KV_RT2
#undef KV_RTL
#undef KV_RT
  return (int)hipGetLastError();
}

int kve_group(const int* expert_of, int n_pairs, int E, int bm, int* order, int* tiles, int max_tiles, int* n_tiles, hipStream_t s) {
  if (n_pairs <= 0 || E <= 0 || E > 1024 || bm <= 0 || max_tiles < n_pairs / bm + (E < n_pairs ? E : n_pairs)) return -1;
  const GroupedRows g{order, tiles, tiles + max_tiles, tiles + 2 * max_tiles, n_tiles, max_tiles, 1};
  hipLaunchKernelGGL(group_pairs_kernel, dim3(1), dim3(1024), 0, s, expert_of, n_pairs, E, bm, g);
  return (int)hipGetLastError();
}

// mode (RowsMode) 1: y [pairs][N / 2], x rows by token (row_div = top); 2: y [pairs][N], x rows by token; 0: y [pairs][N], x rows by pair
int kve_rows(const void* w, const void* x, void* y, int f32, int mode, const int* expert_of, int n_pairs, int top, int E, int N, int K, long long ldx, long long ldy, float limit, float slope, float shift, hipStream_t s) {
  if (n_pairs <= 0 || E <= 0 || top <= 0 || N <= 0 || K <= 0 || mode < PLAIN || mode > SQUARED) return -1;
  const ExpertRowsArgs a{expert_of, n_pairs, mode != PLAIN ? top : 1, N, K, ldx, ldy, ExpertGate{limit, slope, shift}};
  if (f32) {
    if ((K & 3) || (ldx & 3) || (mode == GATED && (N & 15))) return -1;
#define KV_EP(M) hipLaunchKernelGGL((expert_pairs_kernel<M>), dim3(n_pairs), dim3(256), 0, s, (const float*)w, (const float*)x, (float*)y, a)
    if (mode == GATED) KV_EP(GATED);
    else if (mode == SQUARED) KV_EP(SQUARED);
    else KV_EP(PLAIN);
#undef KV_EP
  } else {
    if ((N & 31) || (K & 31) || (ldx & 7) || (ldy & 3) || n_pairs / top > 128) return -1;
    const dim3 grid(N / 32, E);
#define KV_ER(M) hipLaunchKernelGGL((expert_rows_kernel<M>), grid, dim3(256), 0, s, (const bf16raw*)w, (const bf16raw*)x, (bf16raw*)y, a)
    if (mode == GATED) KV_ER(GATED);
    else if (mode == SQUARED) KV_ER(SQUARED);
    else KV_ER(PLAIN);
#undef KV_ER
  }
  return (int)hipGetLastError();
}

}  // extern "C"
