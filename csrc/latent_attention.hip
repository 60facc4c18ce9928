// Latent attention on the matrix cores of gfx950 (bf16).  A token caches one latent c (rank RK, padded); head h's key is W_uk[h] c and
// its value W_uv[h] c; a query sees the last `window` positions up to its own (0: all).  RT > 0: a cache row holds RT more elements, a
// rotated key part that all heads share, and a head's query as many; neighbouring elements 2i, 2i + 1 turn together.
//
// Prompts run on expanded keys and values: latent_gather_kernel copies the latents a step's portions see out of their pages into
// consecutive workspace rows, one matrix product expands them for all heads, and latent_prefill_kernel attends over the rows of the
// product.  Single tokens stay in the latent space: (W_uk^T q) . c are the scores (latent_absorb_kernel, one small matrix per head), the
// weighted sum of the latents is one vector per head (latent_decode_kernel: all heads share the latents, which are read once, as keys and
// as values), and W_uv takes it to the head's value (latent_up_kernel, with the head gates).

#include "attn_tiles.h"

#include <utility>

namespace {
using namespace elem;
using namespace attn;

// ---- latents of the step's prompt portions, page by page -> workspace rows [n][rk]; rows nobody needs become zero.  One wave per row.
struct SpanArgs {
  const int* first_row; const int* first_pos; const int* count; int n_seqs;  // per sequence slot (count 0: none)
  const int* block_tables; int max_blocks, bs_shift;
};

__global__ __launch_bounds__(256) void latent_gather_kernel(const bf16raw* __restrict__ cache, bf16raw* __restrict__ ws, SpanArgs a, int n_rows, int rk) {
  const int r = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (r >= n_rows) return;
  int pos = -1, slot = 0;
  for (int s0 = 0; s0 < a.n_seqs; s0 += 64) {  // the sequence whose rows hold r
    const int s = s0 + lane;
    const int d = s < a.n_seqs ? r - a.first_row[s] : -1;
    const bool hit = d >= 0 && d < a.count[s < a.n_seqs ? s : 0];
    const unsigned long long m = __builtin_amdgcn_ballot_w64(hit);
    if (m) {
      const int l = __builtin_ctzll(m);
      slot = s0 + l;
      pos = a.first_pos[slot] + (r - a.first_row[slot]);
      break;
    }
  }
  const int n16 = rk / 8;
  raw16* dst = reinterpret_cast<raw16*>(ws + (long long)r * rk);
  if (pos < 0) {
    const raw16 zero = {0, 0, 0, 0};
    for (int i = lane; i < n16; i += 64) dst[i] = zero;
    return;
  }
  const int page = a.block_tables[(long long)slot * a.max_blocks + (pos >> a.bs_shift)];
  const raw16* src = reinterpret_cast<const raw16*>(cache + (((long long)page << a.bs_shift) + (pos & ((1 << a.bs_shift) - 1))) * rk);
  for (int i = lane; i < n16; i += 64) dst[i] = src[i];
}

// ---- prompts.  Workgroup: a block of up to 128 consecutive queries of one portion x one head, 32 queries per wave; keys in steps of 32
// from the first one any of its queries sees, rows global -> LDS by LDS-DMA (three stages, counted waits, one barrier per step), shared by
// the waves.  A wave sits out the steps none of its queries sees.
struct LatentPrefillArgs {
  const int* blk_row; const int* blk_n; const int* blk_pos; const int* blk_base;  // first row, queries (0 = unused), first position, workspace row of position 0
  int nh, vdim, window;
  long long ldq; int q_off;   // queries: columns q_off + head * DK of the projections
  long long ldkv; int v_off;  // workspace: keys in columns head * DK, values in v_off + head * DV
  int r_off; const bf16raw* kr; long long ldkr;  // rotated parts: queries' in columns r_off + head * RT of the projections, keys' in rows of their own
  float scale_log2e, out_scale;
  long long ld_gate; int gate_off, gate_each;
  long long ldo; int o_off;
};

// the output gate's factor of element d of a head
__device__ inline float head_gate(const bf16raw* gate_row, int head, int vdim, int each, int d) { return sigmoid(bf2f(gate_row[each ? head * vdim + d : head])); }

template <int DK, int DV, int RT>
__global__ __launch_bounds__(256) void latent_prefill_kernel(const bf16raw* __restrict__ proj, const bf16raw* __restrict__ kv, bf16raw* __restrict__ out, LatentPrefillArgs a) {
  constexpr int NW = 4;
  constexpr int KCH = DK / 8, VCH = DV / 8;        // 16-byte pieces per row
  constexpr int KIT = 32 * KCH / 64 / NW, VIT = 32 * VCH / 64 / NW;  // wave-level pieces (64 x 16 bytes) per wave and step
  static_assert(KIT >= 1 && VIT >= 1 && (RT == 0 || RT == 64), "every wave stages the same number of pieces");
  constexpr int KT = 32 * DK, VT = 32 * DV, ET = 32 * RT;  // elements per image
  constexpr int RIT = RT / 64;                             // pieces of the rotated part per wave and step
  extern __shared__ __attribute__((aligned(16))) bf16raw pf_lds[];  // three stages of K, then of V, then of the rotated part
  const int b = gridDim.y - 1 - blockIdx.y, head = blockIdx.x;  // (heads fastest: a head's keys stay with one XCD; the last blocks of a prompt see the most keys: they start first)
  const int nq = a.blk_n[b];
  if (nq == 0) return;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int lr = lane & 31, hi = lane >> 5;
  const int row0 = a.blk_row[b], pos0 = a.blk_pos[b], base = a.blk_base[b];
  const int last = pos0 + nq - 1;
  auto first_key = [&](int p) { return a.window > 0 && p >= a.window ? p - a.window + 1 : 0; };
  const int first = first_key(pos0);
  const int w0 = 32 * wave;
  const bool on = w0 < nq;
  const int qi = w0 + lr < nq ? w0 + lr : nq - 1;
  const int qpos = pos0 + qi, q_first = first_key(qpos);
  const int w_pos = pos0 + w0, w_last = w_pos + 31 < last ? w_pos + 31 : last;  // the wave's queries (on)
  const int w_first = first_key(w_pos), w_last_first = first_key(w_last);

  frag_ab qa[DK / 16];
  {
    const bf16raw* qp = proj + (long long)(row0 + qi) * a.ldq + a.q_off + head * DK + hi * 8;
#pragma unroll
    for (int ks = 0; ks < DK / 16; ++ks) qa[ks] = *reinterpret_cast<const frag_ab*>(qp + ks * 16);
  }
  frag_ab qr[RT / 16 + 1];
  if constexpr (RT > 0) {
    const bf16raw* qp = proj + (long long)(row0 + qi) * a.ldq + a.r_off + head * RT + hi * 8;
#pragma unroll
    for (int ks = 0; ks < RT / 16; ++ks) qr[ks] = *reinterpret_cast<const frag_ab*>(qp + ks * 16);
  }
  frag_acc o[DV / 32];
#pragma unroll
  for (int n = 0; n < DV / 32; ++n)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[n][r] = 0.f;
  float m_run = -1e30f, l_run = 0.f;

  // rows past the last key read it again (every step issues the same number of pieces); they are masked
  const bf16raw* kp = kv + (long long)base * a.ldkv + head * DK;
  const bf16raw* vp = kv + (long long)base * a.ldkv + a.v_off + head * DV;
  auto stage = [&](int kb, int buf) __attribute__((always_inline)) {
#pragma unroll
    for (int it = 0; it < KIT; ++it) {
      const int p = wave + NW * it, r = p * (64 / KCH) + lane / KCH, c = (lane % KCH) ^ k_swz<DK>(r);
      const int key = kb + r < last ? kb + r : last;
      __builtin_amdgcn_global_load_lds((glb_void*)(kp + (long long)key * a.ldkv + c * 8), (lds_void*)(pf_lds + buf * KT + p * 512), 16, 0, 0);
    }
#pragma unroll
    for (int it = 0; it < VIT; ++it) {
      const int p = wave + NW * it, r = p * (64 / VCH) + lane / VCH, c = (lane % VCH) ^ v_swz<DV>(r);
      const int key = kb + r < last ? kb + r : last;
      __builtin_amdgcn_global_load_lds((glb_void*)(vp + (long long)key * a.ldkv + c * 8), (lds_void*)(pf_lds + 3 * KT + buf * VT + p * 512), 16, 0, 0);
    }
    if constexpr (RT > 0) {
      const int r = wave * 8 + lane / 8, c = (lane & 7) ^ k_swz<64>(r);
      const int key = kb + r < last ? kb + r : last;
      __builtin_amdgcn_global_load_lds((glb_void*)(a.kr + (long long)(base + key) * a.ldkr + c * 8), (lds_void*)(pf_lds + 3 * (KT + VT) + buf * ET + wave * 512), 16, 0, 0);
    }
  };
  stage(first, 0);
  stage(first + 32, 1);
  int buf = 0, ahead = 2;
  for (int kb = first; kb <= last; kb += 32, buf = buf == 2 ? 0 : buf + 1, ahead = ahead == 2 ? 0 : ahead + 1) {
    asm volatile("s_waitcnt vmcnt(%0)" ::"n"(KIT + VIT + RIT) : "memory");  // (the youngest stage may still be on its way)
    __builtin_amdgcn_s_barrier();  // this step's rows have landed; every wave is done with the stage before
    stage(kb + 64, ahead);
    if (!on || kb > w_last || kb + 31 < w_first) continue;
    const bool edge = kb + 31 > w_pos || kb < w_last_first;
    frag_acc st = no_scores();
    if constexpr (RT > 0) {
      const bf16raw* img = pf_lds + 3 * (KT + VT) + buf * ET;
#pragma unroll
      for (int ks = 0; ks < RT / 16; ++ks) {
        const frag_ab kf = *reinterpret_cast<const frag_ab*>(&img[lr * RT + (((2 * ks + hi) ^ k_swz<64>(lr)) << 3)]);
        st = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qr[ks], st, 0, 0, 0);
      }
    }
    attend_tile<DK, DV>(pf_lds + buf * KT, pf_lds + 3 * KT + buf * VT, qa, o, m_run, l_run, a.scale_log2e, edge, qpos - kb, q_first - kb, st);
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // no piece may be in flight when the workgroup gives its LDS back
  const float l = l_run + __shfl_xor(l_run, 32, 64);
  if (!on || w0 + lr >= nq) return;
  const long long row = row0 + qi;
  const bf16raw* gate = proj + row * a.ld_gate + a.gate_off;
  float f = a.out_scale / l;
  if (!a.gate_each) f *= head_gate(gate, head, a.vdim, 0, 0);
  bf16raw* op = out + row * a.ldo + a.o_off + (long long)head * a.vdim;
  const bool vec = (a.vdim & 3) == 0 && (a.ldo & 3) == 0 && (a.o_off & 3) == 0;
#pragma unroll
  for (int n = 0; n < DV / 32; ++n)
#pragma unroll
    for (int rr = 0; rr < 4; ++rr) {
      const int d = 32 * n + 8 * rr + 4 * hi;  // dims d .. d + 3 of this query
      if (d >= a.vdim) continue;
      float4 v = make_float4(o[n][4 * rr] * f, o[n][4 * rr + 1] * f, o[n][4 * rr + 2] * f, o[n][4 * rr + 3] * f);
      if (a.gate_each) {
        const int top = a.vdim - 1;
        v.x *= head_gate(gate, head, a.vdim, 1, d);
        v.y *= head_gate(gate, head, a.vdim, 1, d + 1 < top ? d + 1 : top);
        v.z *= head_gate(gate, head, a.vdim, 1, d + 2 < top ? d + 2 : top);
        v.w *= head_gate(gate, head, a.vdim, 1, d + 3 < top ? d + 3 : top);
      }
      if (vec) {
        if (d < a.vdim) st4(op + d, v);
      } else {
        if (d < a.vdim) st(op + d, v.x);
        if (d + 1 < a.vdim) st(op + d + 1, v.y);
        if (d + 2 < a.vdim) st(op + d + 2, v.z);
        if (d + 3 < a.vdim) st(op + d + 3, v.w);
      }
    }
}

// ---- single tokens, first part: q' = W_uk[h]^T q for the listed rows, [rows][heads][RK].  Workgroup: 64 latent dimensions of one head x 16
// rows.  WRITE: the workgroups behind the last head norm the rows' latents and write them into the cache.  With a rotated part, q' rows are
// RK + RT long; `turn`: the projections' rotated parts have not been rotated yet.
struct LatentRowsArgs {
  const int* rows; int n_rows; const int* slots;
  long long ldp; int q_off, c_off, gate_off, gate_each;
  int nh, rank;
  const float* c_norm; float eps;
  const int* positions; int r_off, kr_off, rot, turn;
  const float* cos_t; const float* sin_t;  // [positions][rot / 2]
};

// the pair 2p, 2p + 1 of a rotated part, for a token at position pos (zero behind it)
__device__ inline float2 turned(const bf16raw* part, int p, int pos, const LatentRowsArgs& a, bool turn) {
  const int half = a.rot >> 1;
  if (p >= half) return make_float2(0.f, 0.f);
  const float x = bf2f(part[2 * p]), y = bf2f(part[2 * p + 1]);
  if (!turn) return make_float2(x, y);
  const float c = a.cos_t[(long long)pos * half + p], s = a.sin_t[(long long)pos * half + p];
  return make_float2(x * c - y * s, y * c + x * s);
}

template <int RK, int DK, int RT, bool WRITE>
__global__ __launch_bounds__(256) void latent_absorb_kernel(const bf16raw* __restrict__ proj, const bf16raw* __restrict__ w, bf16raw* __restrict__ q_lat, bf16raw* __restrict__ cache, LatentRowsArgs a) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, lr = lane & 15, lq = lane >> 4;
  const int h = blockIdx.x, rt = blockIdx.z * 16;
  constexpr int KD = RK + RT;
  if (WRITE && h == a.nh) {
    constexpr int E = RK / 64;
    for (int i = blockIdx.y * 4 + wave; i < 16; i += gridDim.y * 4) {
      if (rt + i >= a.n_rows) return;
      const int t = a.rows[rt + i];
      const int slot = t < 0 ? -1 : a.slots[t];
      if (slot < 0) continue;
      const bf16raw* src = proj + (long long)t * a.ldp + a.c_off + lane * E;
      float v[E], ss = 0.f;
#pragma unroll
      for (int e = 0; e < E; ++e) { v[e] = bf2f(src[e]); ss += v[e] * v[e]; }
      const float rs = 1.f / sqrtf(wave_sum(ss) / (float)a.rank + a.eps);
#pragma unroll
      for (int e = 0; e < E; ++e) cache[(long long)slot * KD + lane * E + e] = f2bf(v[e] * rs * a.c_norm[lane * E + e]);
      if (RT > 0 && lane < RT / 2) {
        const float2 k = turned(proj + (long long)t * a.ldp + a.kr_off, lane, a.positions[t], a, true);
        cache[(long long)slot * KD + RK + 2 * lane] = f2bf(k.x);
        cache[(long long)slot * KD + RK + 2 * lane + 1] = f2bf(k.y);
      }
    }
    return;
  }
  if (RT > 0 && blockIdx.y == 0) {  // the queries' rotated parts, four elements a thread
    const int i = threadIdx.x >> 4, d = (threadIdx.x & 15) * 4;
    const int t = rt + i < a.n_rows ? a.rows[rt + i] : -1;
    if (t >= 0 && a.slots[t] >= 0) {
      const bf16raw* q = proj + (long long)t * a.ldp + a.r_off + h * RT;
      const float2 x = turned(q, d / 2, a.positions[t], a, a.turn), y = turned(q, d / 2 + 1, a.positions[t], a, a.turn);
      st4(q_lat + ((long long)(rt + i) * a.nh + h) * KD + RK + d, make_float4(x.x, x.y, y.x, y.y));
    }
  }
  const int n0 = blockIdx.y * 64 + wave * 16;
  const frag_ab* wp = reinterpret_cast<const frag_ab*>(w) + ((long long)(h * RK + n0) / 16 * (DK / 32)) * 64 + lane;
  const int r = rt + lr;
  const int t = r < a.n_rows ? a.rows[r] : -1;
  const bf16raw* qp = proj + (long long)(t < 0 ? 0 : t) * a.ldp + a.q_off + h * DK + lq * 8;
  frag_acc4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int ks = 0; ks < DK / 32; ++ks) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wp[ks * 64], *reinterpret_cast<const frag_ab*>(qp + ks * 32), acc, 0, 0, 0);
  if (t >= 0) st4(q_lat + ((long long)r * a.nh + h) * KD + n0 + 4 * lq, make_float4(acc[0], acc[1], acc[2], acc[3]));
}

// ---- second part: attention in the latent space.  grid (listed rows, groups of 16 heads, shares): the keys a row sees, in blocks of 16
// dealt out to the waves of its workgroups.  A wave copies a block of latents into LDS of its own (LDS-DMA, two buffers), multiplies them
// as A operand with the 16 heads' q' (S^T: a lane owns one head and 4 keys), and the weights, already in the A layout of
// mfma_f32_16x16x16_bf16, with the same latents again, read transposed.  A rotated part (RT) lies behind the block's latents, rows of 128
// bytes whose pieces are swizzled by pairs of rows, and only enters the scores.
struct LatentDecodeArgs {
  const int* block_tables; int max_blocks;
  const int* rows; const int* tok_seq; const int* positions; const int* slots;
  int nh, bs_shift, window, shares;
  float scale_log2e;
};

__device__ inline int lat_swz(int row) { return ((row & 7) << 1) | ((row >> 3) & 1); }  // sixteen distinct pieces over 16 rows; even ones over any eight

template <int... I>
__device__ inline void latent_key_reads(raw16 (&kf)[sizeof...(I)], const unsigned int (&at)[4], std::integer_sequence<int, I...>) {
  ((kf[I] = lds_read16_at<(I >> 2) * 256>(at[I & 3])), ...);
}

// out: bf16 [rows][heads][RK] normalised (shares 1), or fp32 [rows][heads][shares][RK + 4]: maximum, sum, -, -, unnormalised sum
template <int RK, int RT, bool SPLIT>
__global__ __launch_bounds__(256) void latent_decode_kernel(const bf16raw* __restrict__ q_lat, const bf16raw* __restrict__ cache, void* __restrict__ out, LatentDecodeArgs a) {
  constexpr int NW = 4;
  constexpr int PC = RK / 8, PIECES = 16 * PC / 64, RPP = 64 / PC;  // 16-byte pieces per latent; wave-level pieces per block; rows per wave-level piece
  constexpr int KD = RK + RT, NR = RT / 32;  // cache row; fragments (and wave-level pieces) of a block's rotated part
  constexpr int BLK = 16 * RK, BUF = 16 * KD;
  extern __shared__ __attribute__((aligned(16))) bf16raw ld_lds[];  // per wave two blocks, later its output (fp32 [16][RK])
  __shared__ float ml[NW][16][2];
  const int r_list = blockIdx.x, t = a.rows[r_list];
  if (t < 0 || a.slots[t] < 0) return;  // unused entry, or a padding row: it has no place in the cache
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63;
  const int lr = lane & 15, lq = lane >> 4;
  const int h0 = blockIdx.y * 16;
  const int nhd = a.nh - h0 < 16 ? a.nh - h0 : 16;
  const int pos = a.positions[t];
  const int first = a.window > 0 && pos >= a.window ? pos - a.window + 1 : 0;
  const int b0 = first >> 4, nb = (pos >> 4) - b0 + 1;  // blocks of 16 keys; each holds a visible one
  const int stride = a.shares * NW, me = blockIdx.z * NW + wave;
  scalar_int* bt = (scalar_int*)(uintptr_t)(a.block_tables + (long long)a.tok_seq[t] * a.max_blocks);  // (constant during the kernel)
  const int bs_mask = (1 << a.bs_shift) - 1;

  frag_ab qb[RK / 32], qr[NR + 1];
  {
    const bf16raw* qp = q_lat + ((long long)r_list * a.nh + h0 + (lr < nhd ? lr : nhd - 1)) * KD + lq * 8;
#pragma unroll
    for (int ks = 0; ks < RK / 32; ++ks) qb[ks] = *reinterpret_cast<const frag_ab*>(qp + ks * 32);
#pragma unroll
    for (int ks = 0; ks < NR; ++ks) qr[ks] = *reinterpret_cast<const frag_ab*>(qp + RK + ks * 32);
  }
  bf16raw* mine = ld_lds + wave * 2 * BUF;
  auto rot_swz = [](int row) { return (row >> 1) & 7; };
  unsigned int rot_piece[NR + 1];
#pragma unroll
  for (int p = 0; p < NR; ++p) {
    const int r = p * 8 + lane / 8;
    rot_piece[p] = (unsigned int)(r * KD + RK + ((lane & 7) ^ rot_swz(r)) * 8) * 2;
  }
  unsigned int piece[PIECES];  // byte offsets of the lane's pieces inside a block
#pragma unroll
  for (int p = 0; p < PIECES; ++p) {
    const int r = p * RPP + lane / PC;
    piece[p] = (unsigned int)(r * KD + ((lane % PC) ^ lat_swz(r)) * 8) * 2;
  }
  auto stage = [&](int b, int buf) __attribute__((always_inline)) {
    const int key = (b0 + b) << 4;
    const char* src = reinterpret_cast<const char*>(cache + (((long long)bt[key >> a.bs_shift] << a.bs_shift) + (key & bs_mask)) * KD);
#pragma unroll
    for (int p = 0; p < PIECES; ++p) {
      unsigned int off = piece[p];
      asm volatile("" : "+v"(off));  // (a scalar base and a 32-bit lane offset: no 64-bit sums per piece)
      __builtin_amdgcn_global_load_lds((glb_void*)(src + off), (lds_void*)(mine + buf * BUF + p * 512), 16, 0, 0);
    }
#pragma unroll
    for (int p = 0; p < NR; ++p) {
      unsigned int off = rot_piece[p];
      asm volatile("" : "+v"(off));
      __builtin_amdgcn_global_load_lds((glb_void*)(src + off), (lds_void*)(mine + buf * BUF + BLK + p * 512), 16, 0, 0);
    }
  };
  // LDS addresses of the lane's fragments in buffer 0.  A piece's place is its number XOR the row's swizzle (four bits): what lies beyond
  // sixteen pieces is a constant offset.
  const unsigned int lds0 = (unsigned int)(uintptr_t)(lds_void*)mine;
  const int vr = 4 * lq + (lr >> 2);
  unsigned int k_at[4], v_at[8], r_at[NR + 1];
#pragma unroll
  for (int j = 0; j < NR; ++j) r_at[j] = lds0 + (BLK + lr * RT + (((4 * j + lq) ^ rot_swz(lr)) << 3)) * 2;
#pragma unroll
  for (int j = 0; j < 4; ++j) k_at[j] = lds0 + (lr * RK + (((4 * j + lq) ^ lat_swz(lr)) << 3)) * 2;
#pragma unroll
  for (int j = 0; j < 8; ++j) v_at[j] = lds0 + (vr * RK + (((2 * j + ((lr & 3) >> 1)) ^ lat_swz(vr)) << 3) + (lr & 1) * 4) * 2;

  frag_acc4 o[RK / 16];
#pragma unroll
  for (int n = 0; n < RK / 16; ++n) o[n] = (frag_acc4){0.f, 0.f, 0.f, 0.f};
  float m_run = -1e30f, l_run = 0.f;
  if (me < nb) stage(me, 0);
  int b = me;
  unsigned int flip = 0;  // byte offset of the block's buffer
  bool staged = false;    // the next block is on its way already
  // The reference m_run of the exponentials is the first block's maximum and follows only when a later one outgrows it by 2^24 (weights
  // and sums are floating point: their precision does not depend on it).  Then the inner loop is left, the sums are rescaled and the
  // block is taken up again: inside the loop only matrix instructions touch the sums, so they stay in accumulation registers.
  while (b < nb) {
    float mx;
    bool outgrown = false;
    for (; b < nb; b += stride, flip ^= BUF * 2, staged = false) {
      if (b + stride < nb) {
        if (!staged) stage(b + stride, flip ? 0 : 1);
        asm volatile("s_waitcnt vmcnt(%0)" ::"n"(PIECES + NR) : "memory");
      } else {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
      }
      constexpr int NK = RK / 32, KG = NK < 8 ? NK : 8;  // key fragments; as many are in flight ahead of their products
      raw16 kf[NK], rf[NR + 1];
#pragma unroll
      for (int j = 0; j < NR; ++j) rf[j] = lds_read16_at<0>(r_at[j] + flip);
      {
        unsigned int at[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) at[j] = k_at[j] + flip;
        latent_key_reads(kf, at, std::make_integer_sequence<int, NK>{});
      }
      frag_acc4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = s0;
#pragma unroll
      for (int g = 0; g < NK / KG; ++g) {
        asm volatile("s_waitcnt lgkmcnt(%0)" ::"n"(NK - KG * (g + 1)) : "memory");
#pragma unroll
        for (int i = g * KG; i < (g + 1) * KG; ++i) asm volatile("" : "+v"(kf[i]));  // (uses stay behind the wait)
        if (g == 0) {  // (read ahead of the others: landed as well)
#pragma unroll
          for (int j = 0; j < NR; ++j) {
            asm volatile("" : "+v"(rf[j]));
            (j & 1 ? s1 : s0) = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(frag_ab, rf[j]), qr[j], j & 1 ? s1 : s0, 0, 0, 0);
          }
        }
#pragma unroll
        for (int i = g * KG; i < (g + 1) * KG; i += 2) {
          s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(frag_ab, kf[i]), qb[i], s0, 0, 0, 0);
          s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(frag_ab, kf[i + 1]), qb[i + 1], s1, 0, 0, 0);
        }
      }
      constexpr int G = 8;  // transposed reads in flight ahead of their products; the first ones run under the softmax
      tr_b64 va[2][G];
      unsigned int at[G];
#pragma unroll
      for (int i = 0; i < G; ++i) at[i] = v_at[i] + flip;
      auto v_read = [&](auto g_) __attribute__((always_inline)) {
        constexpr int g = decltype(g_)::value;
#pragma unroll
        for (int i = 0; i < G; ++i) va[g & 1][i] = lds_read_tr_at<g * 256>(at[i]);
      };
      v_read(std::integral_constant<int, 0>{});
      const frag_acc4 st = s0 + s1;
      const int k0 = ((b0 + b) << 4) + 4 * lq;
      float sc[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) sc[r] = (k0 + r >= first && k0 + r <= pos) ? st[r] * a.scale_log2e : -1e30f;
      mx = fmaxf(fmaxf(sc[0], sc[1]), fmaxf(sc[2], sc[3]));
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      if (b == me && !staged) m_run = mx;
      if (__builtin_amdgcn_ballot_w64(mx > m_run + 24.f) != 0) {
        lds_landed(va[0]);
        outgrown = true;
        break;
      }
      typedef __attribute__((ext_vector_type(4))) __bf16 bf4;
      bf4 pb;
      float psum = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float p = __builtin_amdgcn_exp2f(sc[r] - m_run);
        psum += p;
        pb[r] = (__bf16)p;
      }
      l_run += psum;
      const frag_b64 pa = __builtin_bit_cast(frag_b64, pb);
      auto v_group = [&](auto g_) __attribute__((always_inline)) {
        constexpr int g = decltype(g_)::value;
        if constexpr (g < RK / 16 / G) {
          lds_landed(va[g & 1]);
          if constexpr (g + 1 < RK / 16 / G) v_read(std::integral_constant<int, g + 1>{});
#pragma unroll
          for (int i = 0; i < G; ++i) o[g * G + i] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(pa, __builtin_bit_cast(frag_b64, va[g & 1][i]), o[g * G + i], 0, 0, 0);
        }
      };
      v_group(std::integral_constant<int, 0>{});
      v_group(std::integral_constant<int, 1>{});
      v_group(std::integral_constant<int, 2>{});
      v_group(std::integral_constant<int, 3>{});
    }
    if (!outgrown) break;
    const float m_new = mx > m_run + 24.f ? mx : m_run;
    const float corr = __builtin_amdgcn_exp2f(m_run - m_new);
    m_run = m_new;
    l_run *= corr;
    staged = true;
    float cr[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) cr[r] = __shfl(corr, 4 * lq + r, 64);  // output rows are heads 4 lq + r
#pragma unroll
    for (int n = 0; n < RK / 16; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) o[n][r] *= cr[r];
  }
  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  if (lq == 0) { ml[wave][lr][0] = m_run; ml[wave][lr][1] = l_run; }
  float* os = reinterpret_cast<float*>(mine);  // (the wave's own LDS: its reads above are done, nothing is in flight)
#pragma unroll
  for (int r = 0; r < 4; ++r)
#pragma unroll
    for (int n = 0; n < RK / 16; ++n) os[(4 * lq + r) * RK + 16 * n + lr] = o[n][r];
  __syncthreads();
  const float* oa = reinterpret_cast<const float*>(ld_lds);
  for (int i = tid; i < nhd * (RK / 4); i += 256) {
    const int h = i / (RK / 4), d = (i % (RK / 4)) * 4;
    float m = ml[0][h][0];
#pragma unroll
    for (int w = 1; w < NW; ++w) m = fmaxf(m, ml[w][h][0]);
    float l = 0.f;
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      const float c = __builtin_amdgcn_exp2f(ml[w][h][0] - m);
      const float4 x = ld4(oa + w * BUF + h * RK + d);
      l += c * ml[w][h][1];
      v.x += c * x.x; v.y += c * x.y; v.z += c * x.z; v.w += c * x.w;
    }
    const long long row = (long long)r_list * a.nh + h0 + h;
    if constexpr (SPLIT) {
      float* p = reinterpret_cast<float*>(out) + (row * a.shares + blockIdx.z) * (RK + 4);
      st4(p + 4 + d, v);
      if (d == 0) { p[0] = m; p[1] = l; }
    } else {
      const float f = 1.f / l;
      st4(reinterpret_cast<bf16raw*>(out) + row * RK + d, make_float4(v.x * f, v.y * f, v.z * f, v.w * f));
    }
  }
}

// ---- with shares: their partial sums [rows][heads][shares][RK + 4] -> bf16 [rows][heads][RK].  One wave per row and head.
template <int RK>
__global__ __launch_bounds__(64) void latent_combine_kernel(const float* __restrict__ part, bf16raw* __restrict__ lat, const int* __restrict__ rows, const int* __restrict__ slots, int nh, int shares) {
  constexpr int E = RK / 64;  // elements per lane
  const int t = rows[blockIdx.x], lane = threadIdx.x;
  if (t < 0 || slots[t] < 0) return;
  const long long row = (long long)blockIdx.x * nh + blockIdx.y;
  const float* p = part + row * shares * (RK + 4);
  const bool on = lane < shares;  // (at most 64)
  const float m = on ? p[(long long)lane * (RK + 4)] : -1e30f;
  const float top = wave_max(m);
  const float f = on ? __builtin_amdgcn_exp2f(m - top) : 0.f;
  const float l = wave_sum(on ? f * p[(long long)lane * (RK + 4) + 1] : 0.f);
  const float w = f / l;
  float v[E];
#pragma unroll
  for (int e = 0; e < E; ++e) v[e] = 0.f;
#pragma unroll 4
  for (int s = 0; s < shares; ++s) {
    const float ws = __shfl(w, s, 64);
    const float* x = p + (long long)s * (RK + 4) + 4 + lane * E;
#pragma unroll
    for (int e = 0; e < E; e += 2) {
      const float2 y = *reinterpret_cast<const float2*>(x + e);
      v[e] += ws * y.x;
      v[e + 1] += ws * y.y;
    }
  }
#pragma unroll
  for (int e = 0; e < E; ++e) lat[row * RK + lane * E + e] = f2bf(v[e]);
}

// ---- third part: value = W_uv[h] (weighted latent), times out_scale and the head's gate.  Workgroup: one head x 16 listed rows x
// DV / gridDim.z features.
struct LatentUpArgs {
  LatentRowsArgs r;
  int vdim;
  float out_scale;
  long long ldo; int o_off;
};

template <int RK, int DV>
__global__ __launch_bounds__(256) void latent_up_kernel(const bf16raw* __restrict__ lat, const bf16raw* __restrict__ w, const bf16raw* __restrict__ proj, bf16raw* __restrict__ out, LatentUpArgs a) {
  constexpr int LS = RK + 8;
  __shared__ __attribute__((aligned(16))) bf16raw x_s[16 * LS];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, lr = lane & 15, lq = lane >> 4;
  const int h = blockIdx.x, rt = blockIdx.y * 16;
#pragma unroll
  for (int i = threadIdx.x; i < 16 * (RK / 8); i += 256) {  // 16 rows x RK into LDS, 8 elements a time
    const int rr = i / (RK / 8), c = (i % (RK / 8)) * 8, r = rt + rr;
    const int t = r < a.r.n_rows ? a.r.rows[r] : -1;
    raw16 v = {0, 0, 0, 0};
    if (t >= 0 && a.r.slots[t] >= 0) v = *reinterpret_cast<const raw16*>(lat + ((long long)r * a.r.nh + h) * RK + c);
    *reinterpret_cast<raw16*>(x_s + rr * LS + c) = v;
  }
  __syncthreads();
  const int r = rt + lr;
  const int t = r < a.r.n_rows ? a.r.rows[r] : -1;
  const bool live = t >= 0 && a.r.slots[t] >= 0;
  const bf16raw* gate = proj + (long long)(live ? t : 0) * a.r.ldp + a.r.gate_off;
  float f = a.out_scale;
  if (live && !a.r.gate_each) f *= head_gate(gate, h, a.vdim, 0, 0);
  const bool vec = (a.vdim & 3) == 0 && (a.ldo & 3) == 0 && (a.o_off & 3) == 0;
  bf16raw* op = out + (long long)(t < 0 ? 0 : t) * a.ldo + a.o_off + (long long)h * a.vdim;
  for (int n = blockIdx.z * 4 + wave; n < DV / 16; n += 4 * gridDim.z) {
    const frag_ab* wp = reinterpret_cast<const frag_ab*>(w) + ((long long)(h * DV + 16 * n) / 16 * (RK / 32)) * 64 + lane;
    frag_acc4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < RK / 32; ++ks) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wp[ks * 64], *reinterpret_cast<const frag_ab*>(&x_s[lr * LS + ks * 32 + lq * 8]), acc, 0, 0, 0);
    if (!live) continue;
    const int d = 16 * n + 4 * lq;
    if (d >= a.vdim) continue;
#pragma unroll
    for (int e = 0; e < 4; ++e) acc[e] *= a.r.gate_each ? f * head_gate(gate, h, a.vdim, 1, d + e < a.vdim ? d + e : d) : f;
    if (vec) {
      st4(op + d, make_float4(acc[0], acc[1], acc[2], acc[3]));
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (d + e < a.vdim) st(op + d + e, acc[e]);
    }
  }
}

bool pow2(int n) { return n > 0 && (n & (n - 1)) == 0; }
int log2i(int n) { int s = 0; while ((1 << s) < n) ++s; return s; }

}  // namespace

extern "C" {

// padded sizes the kernels are built for
int kvl_supported(int dkp, int dvp, int rk) { return (dkp == 64 || dkp == 128 || dkp == 256) && (dvp == 64 || dvp == 128 || dvp == 256) && (rk == 128 || rk == 256 || rk == 512); }

int kvl_gather(const void* cache, void* ws, const int* first_row, const int* first_pos, const int* count, int n_seqs, const int* block_tables, int max_blocks, int block_size, int n_rows, int rk,
               hipStream_t s) {
  if (n_rows <= 0 || n_seqs <= 0 || rk <= 0 || (rk & 7) || !pow2(block_size)) return -1;
  const SpanArgs a{first_row, first_pos, count, n_seqs, block_tables, max_blocks, log2i(block_size)};
  hipLaunchKernelGGL(latent_gather_kernel, dim3((n_rows + 3) / 4), dim3(256), 0, s, (const bf16raw*)cache, (bf16raw*)ws, a, n_rows, rk);
  return (int)hipGetLastError();
}

// rt: elements of the rotated part (0, or 64 with rows kr [.., ldkr] of the keys' parts, indexed like those of kv)
int kvl_prefill(const void* proj, long long ldp, int q_off, int r_off, int gate_off, int gate_each, const void* kv, long long ldkv, int v_off, const void* kr, long long ldkr, int rt, const int* blocks,
                int block_stride, int n_blocks, void* out, long long ldo, int o_off, int nh, int dkp, int vdim, int dvp, int window, float scale, float out_scale, hipStream_t s) {
  if (n_blocks <= 0 || n_blocks > block_stride || nh <= 0 || vdim <= 0 || vdim > dvp || window < 0 || !kvl_supported(dkp, dvp, 128) || (ldp & 7) || (q_off & 7) || (ldkv & 7) || (v_off & 7) ||
      (rt != 0 && (rt != 64 || !kr || (ldkr & 7) || (r_off & 7) || ((uintptr_t)kr & 15))))
    return -1;
  const LatentPrefillArgs a{blocks, blocks + block_stride, blocks + 2 * block_stride, blocks + 3 * block_stride, nh, vdim, window, ldp, q_off, ldkv, v_off, r_off, (const bf16raw*)kr, ldkr,
                            scale * 1.4426950408889634f, out_scale, ldp, gate_off, gate_each, ldo, o_off};
#define KV_LP(DK, DV, RT)                                                                                                                                                       \
  do {                                                                                                                                                                          \
    constexpr size_t lds = (size_t)3 * 32 * (DK + DV + RT) * sizeof(bf16raw);                                                                                                   \
    if (lds > 65536 && hipFuncSetAttribute((const void*)latent_prefill_kernel<DK, DV, RT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) return -1;       \
    hipLaunchKernelGGL((latent_prefill_kernel<DK, DV, RT>), dim3(nh, n_blocks), dim3(256), lds, s, (const bf16raw*)proj, (const bf16raw*)kv, (bf16raw*)out, a);                  \
  } while (0)
#define KV_LPR(DK, DV) do { if (rt) KV_LP(DK, DV, 64); else KV_LP(DK, DV, 0); } while (0)
#define KV_LPV(DK) do { if (dvp == 64) KV_LPR(DK, 64); else if (dvp == 128) KV_LPR(DK, 128); else KV_LPR(DK, 256); } while (0)
  if (dkp == 64) KV_LPV(64);
  else if (dkp == 128) KV_LPV(128);
  else KV_LPV(256);
#undef KV_LPV
#undef KV_LPR
#undef KV_LP
  return (int)hipGetLastError();
}

// rows: listed token rows (-1 = unused).  write: the rows' latents go into the cache as well.  q_lat [rows][heads][rk + rt]
int kvl_absorb(const void* proj, long long ldp, int q_off, int c_off, const void* w, void* q_lat, void* cache, int write, const int* rows, int n_rows, const int* slots, const float* c_norm, int rank,
               float eps, int nh, int dkp, int rk, int rt, const int* positions, int r_off, int kr_off, int rot, int turn, const float* cos_t, const float* sin_t, hipStream_t s) {
  if (n_rows <= 0 || nh <= 0 || rank <= 0 || rank > rk || !kvl_supported(dkp, 64, rk) || (ldp & 7) || (q_off & 7) || (c_off & 7) || (write && !c_norm) ||
      (rt != 0 && (rt != 64 || rot <= 0 || rot > rt || (rot & 1) || !positions || !cos_t || !sin_t)))
    return -1;
  const LatentRowsArgs a{rows, n_rows, slots, ldp, q_off, c_off, 0, 0, nh, rank, c_norm, eps, positions, r_off, kr_off, rot, turn, cos_t, sin_t};
  const dim3 grid(nh + (write ? 1 : 0), rk / 64, (n_rows + 15) / 16);
#define KV_LA(RK, DK, RT)                                                                                                                                                       \
  do {                                                                                                                                                                          \
    if (write) hipLaunchKernelGGL((latent_absorb_kernel<RK, DK, RT, true>), grid, dim3(256), 0, s, (const bf16raw*)proj, (const bf16raw*)w, (bf16raw*)q_lat, (bf16raw*)cache, a); \
    else hipLaunchKernelGGL((latent_absorb_kernel<RK, DK, RT, false>), grid, dim3(256), 0, s, (const bf16raw*)proj, (const bf16raw*)w, (bf16raw*)q_lat, (bf16raw*)cache, a);      \
  } while (0)
#define KV_LAR(RK, DK) do { if (rt) KV_LA(RK, DK, 64); else KV_LA(RK, DK, 0); } while (0)
#define KV_LAK(RK) do { if (dkp == 64) KV_LAR(RK, 64); else if (dkp == 128) KV_LAR(RK, 128); else KV_LAR(RK, 256); } while (0)
  if (rk == 128) KV_LAK(128);
  else if (rk == 256) KV_LAK(256);
  else KV_LAK(512);
#undef KV_LAK
#undef KV_LAR
#undef KV_LA
  return (int)hipGetLastError();
}

// lat: bf16 [rows][heads][rk]; part (shares > 1): fp32 [rows][heads][shares][rk + 4]
int kvl_decode(const void* q_lat, const void* cache, void* lat, float* part, const int* block_tables, int max_blocks, const int* rows, int n_rows, const int* tok_seq, const int* positions, const int* slots,
               int nh, int rk, int rt, int block_size, int window, float scale, int shares, hipStream_t s) {
  if (n_rows <= 0 || nh <= 0 || !kvl_supported(64, 64, rk) || !pow2(block_size) || block_size < 16 || window < 0 || shares < 1 || shares > 64 || (shares > 1 && !part) || (rt != 0 && rt != 64)) return -1;
  const LatentDecodeArgs a{block_tables, max_blocks, rows, tok_seq, positions, slots, nh, log2i(block_size), window, shares, scale * 1.4426950408889634f};
#define KV_LD(RK, RT, SP)                                                                                                                                                     \
  do {                                                                                                                                                                        \
    constexpr size_t lds = (size_t)4 * 2 * 16 * (RK + RT) * sizeof(bf16raw);                                                                                                  \
    if (lds > 65536 && hipFuncSetAttribute((const void*)latent_decode_kernel<RK, RT, SP>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) return -1;      \
    hipLaunchKernelGGL((latent_decode_kernel<RK, RT, SP>), dim3(n_rows, (nh + 15) / 16, shares), dim3(256), lds, s, (const bf16raw*)q_lat, (const bf16raw*)cache, SP ? (void*)part : lat, a); \
  } while (0)
#define KV_LDR(RK, SP) do { if (rt) KV_LD(RK, 64, SP); else KV_LD(RK, 0, SP); } while (0)
#define KV_LD2(RK)                                                                                                                                             \
  do {                                                                                                                                                         \
    if (shares == 1) { KV_LDR(RK, false); break; }                                                                                                             \
    KV_LDR(RK, true);                                                                                                                                          \
    hipLaunchKernelGGL((latent_combine_kernel<RK>), dim3(n_rows, nh), dim3(64), 0, s, part, (bf16raw*)lat, rows, slots, nh, shares);                           \
  } while (0)
  if (rk == 128) KV_LD2(128);
  else if (rk == 256) KV_LD2(256);
  else KV_LD2(512);
#undef KV_LD2
#undef KV_LDR
#undef KV_LD
  return (int)hipGetLastError();
}

int kvl_up(const void* lat, const void* w, const void* proj, long long ldp, int gate_off, int gate_each, void* out, long long ldo, int o_off, const int* rows, int n_rows, const int* slots, int nh,
           int rk, int vdim, int dvp, float out_scale, int parts, hipStream_t s) {
  if (n_rows <= 0 || nh <= 0 || vdim <= 0 || vdim > dvp || parts < 1 || !kvl_supported(64, dvp, rk)) return -1;
  const LatentUpArgs a{{rows, n_rows, slots, ldp, 0, 0, gate_off, gate_each, nh, 0, nullptr, 0.f, nullptr, 0, 0, 0, 0, nullptr, nullptr}, vdim, out_scale, ldo, o_off};
  const dim3 grid(nh, (n_rows + 15) / 16, parts);
#define KV_LU(RK, DV) hipLaunchKernelGGL((latent_up_kernel<RK, DV>), grid, dim3(256), 0, s, (const bf16raw*)lat, (const bf16raw*)w, (const bf16raw*)proj, (bf16raw*)out, a)
#define KV_LUV(RK) do { if (dvp == 64) KV_LU(RK, 64); else if (dvp == 128) KV_LU(RK, 128); else KV_LU(RK, 256); } while (0)
  if (rk == 128) KV_LUV(128);
  else if (rk == 256) KV_LUV(256);
  else KV_LUV(512);
#undef KV_LUV
#undef KV_LU
  return (int)hipGetLastError();
}

}  // extern "C"
