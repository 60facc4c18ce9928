// Prompt and decode attention inside chunks or sliding windows of the sequence, on the matrix cores of gfx950: bf16 queries, paged bf16 keys and values with
// their own (padded) head sizes DK and DV, any number of query heads per key head.
//
// A query at position p sees the keys [p - p % chunk, p] (chunk = 0: all keys up to p) or, with a window, the last `window` ones up to p and the
// first `keep` ones of the sequence.  To a scaled score a distance bias may be added (REL), rel[head][distance], its last entry for all that is
// further away; a sink is one more term exp(sink[head]) of the softmax's denominator: running maximum and sum start from it.  Work item: a block of up to 32
// consecutive queries of one portion x the query heads of one key head, one head per wave (NW waves; more heads: grid.z).
// Keys run in aligned steps of 32 from the chunk of the block's first query: K and V rows go global -> LDS by LDS-DMA (16-byte
// pieces, three stages, counted waits, one barrier per step), shared by the waves; the page of a piece is wave-uniform, so its
// number comes through the scalar path and no vector load stands between the DMAs.  As in the other prompt kernels everything is computed transposed:
//   S^T = K Q^T on mfma_f32_32x32x16_bf16 (A = keys, B = queries): a lane owns one query (lane & 31) and 16 of the step's keys;
//   the exponentiated accumulators, packed to bf16, are the B operand of O^T += V^T P^T when the k dimension is read as the
//   permutation slot(8 hi + j) = key 16 s + 8 (j / 4) + 4 hi + j % 4; V^T comes out of LDS by transposed 8-byte reads.
// LDS images are row-major with 16-byte pieces XOR-swizzled by the row (applied to the source address: LDS-DMA writes in lane
// order), so that the rows of a fragment read spread over the banks.
// Where the values are the keys as projected (RT >= 0), the cache holds one row per token and key head, [key, DV | its rotated first
// dimensions, RT], and beside it the fp32 factor that norms the key.  A query is zero in the dimensions that turn and has them, rotated, behind
// the others, so that query . row is the score but for the factor, which multiplies it afterwards; the same row, staged once, is the value.
// Epilogue: 1 / sum, out_scale and the gate: sigmoid(gate[row][head]) (gated 1) or sigmoid(gate[row][head vdim + i]) (2).

#include "attn_tiles.h"

namespace {
using namespace elem;
using namespace attn;

constexpr float LOG2E = 1.4426950408889634f;

// what a query sees, and what its scores get besides
struct Sight { int chunk, window, keep; const float* sink; const float* rel; int rel_n; };
__device__ inline int first_seen(const Sight& s, int pos) { return s.window > 0 ? (pos >= s.window ? pos - s.window + 1 : 0) : s.chunk > 0 ? pos - pos % s.chunk : 0; }

struct ChunkAttnArgs {
  const float* key_scale;  // RT >= 0: [cache rows]
  const int* block_tables; int max_blocks;
  const int* blk_row; const int* blk_n; const int* blk_pos; const int* blk_slot;  // query blocks: first row, queries (0 = unused), first position, block-table row
  int nh, nkv, vdim, bs_shift;
  Sight see;
  float scale_log2e, out_scale;
  long long ld_gate; int gate_off, gated;
  long long ldo; int o_off;
};

template <int DK, int DV, int NW, bool REL, int RT>
__global__ __launch_bounds__(64 * NW, DV <= 128 ? 2 : 1) void chunk_prefill_kernel(const bf16raw* __restrict__ q, const bf16raw* __restrict__ k_cache, const bf16raw* __restrict__ v_cache,
                                                                const bf16raw* __restrict__ gate, bf16raw* __restrict__ out, ChunkAttnArgs a) {
  constexpr bool ONE = RT >= 0;  // one row is key and value; the second image then holds the rotated parts
  static_assert(!ONE || DK == DV, "the values are the keys");
  constexpr int D2 = ONE ? RT : DV, KST = ONE ? DK + RT : DK, VST = ONE ? KST : DV;  // width of the second image; row strides in the cache
  constexpr int KCH = DK / 8, VCH = D2 > 0 ? D2 / 8 : 1;  // 16-byte pieces per row
  constexpr int KP = 32 * KCH / 64, VP = D2 * 32 / 512;   // wave-level pieces (64 x 16 bytes) per step
  constexpr int KIT = (KP + NW - 1) / NW, VIT = (VP + NW - 1) / NW;
  constexpr int KT = 32 * DK, VT = 32 * D2;  // elements per image
  extern __shared__ __attribute__((aligned(16))) bf16raw pf_lds[];  // three stages of K, then of V
  // a step's distance biases (of the wave's head) and keys' factors, three stages: by LDS-DMA like the rest, so that no other load is in flight
  constexpr int AUX = (REL ? 1 : 0) + (ONE ? 1 : 0);
  __shared__ __attribute__((aligned(16))) float aux_s[NW][3][AUX > 0 ? AUX * 64 : 1];
  const int b = gridDim.x - 1 - blockIdx.x, g = blockIdx.y;  // (the last blocks of a prompt see the most keys: they start first)
  const int nq = a.blk_n[b];
  if (nq == 0) return;
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63;
  const int lr = lane & 31, hi = lane >> 5;
  const int rep = a.nh / a.nkv;
  const int hg = blockIdx.z * NW + wave;  // head within the group
  const bool head_on = hg < rep;          // (a wave without a head only stages)
  const int head = g * rep + (head_on ? hg : rep - 1);
  const int row0 = a.blk_row[b], pos0 = a.blk_pos[b];
  scalar_int* bt = (scalar_int*)(uintptr_t)(a.block_tables + (long long)a.blk_slot[b] * a.max_blocks);  // (read through the scalar path: constant during the kernel)
  const int qi = lr < nq ? lr : nq - 1;
  const int qpos = pos0 + qi;
  const int first = first_seen(a.see, pos0);  // first key any query of the block sees (behind the kept ones)
  const int q_first = first_seen(a.see, qpos);
  const int last = pos0 + nq - 1;
  const int last_first = first_seen(a.see, last);  // first key of the last query

  frag_ab qa[DK / 16], qr[RT > 0 ? RT / 16 : 1];
  {
    const bf16raw* qp = q + ((long long)(row0 + qi) * a.nh + head) * KST + hi * 8;
#pragma unroll
    for (int ks = 0; ks < DK / 16; ++ks) qa[ks] = *reinterpret_cast<const frag_ab*>(qp + ks * 16);
    if constexpr (RT > 0) {
#pragma unroll
      for (int ks = 0; ks < RT / 16; ++ks) qr[ks] = *reinterpret_cast<const frag_ab*>(qp + DK + ks * 16);
    }
  }
  frag_acc o[DV / 32];
#pragma unroll
  for (int n = 0; n < DV / 32; ++n)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[n][r] = 0.f;
  float m_run = -1e30f, l_run = 0.f;
  if (a.see.sink) {
    m_run = a.see.sink[head] * LOG2E;
    l_run = hi == 0 ? 1.f : 0.f;  // (the lanes' sums are added up at the end)
  }

  // LDS-DMA of a step: wave-level piece p of an image covers 64 consecutive 16-byte slots, 2 to 8 rows of one page.  Steps past the
  // end read the last page again (every step issues the same number of pieces); rows past the last key are masked.
  const int bs_mask = (1 << a.bs_shift) - 1, last_page = last >> a.bs_shift;
  auto piece_row = [&](int key) -> long long {  // cache row of the (aligned) first row of a piece
    const int pg = key >> a.bs_shift;
    return ((long long)bt[pg < last_page ? pg : last_page] * a.nkv + g) * (bs_mask + 1) + (key & bs_mask);
  };
  // REL: entry e of a step's slice is the distance pos0 + e - 31 - kb; query lr and key k are e = lr + 31 - k
  const float* rel = REL ? a.see.rel + (long long)head * a.see.rel_n : nullptr;
  auto stage = [&](int kb, int buf) __attribute__((always_inline)) {
    if constexpr (REL) {
      int d = pos0 + lane - 31 - kb;
      d = d < 0 ? 0 : d < a.see.rel_n ? d : a.see.rel_n - 1;
      __builtin_amdgcn_global_load_lds((glb_void*)(rel + d), (lds_void*)&aux_s[wave][buf][0], 4, 0, 0);
    }
    if constexpr (ONE) {
      const long long r0 = piece_row(kb), r1 = piece_row(kb + 16);
      __builtin_amdgcn_global_load_lds((glb_void*)(a.key_scale + ((lane & 16) ? r1 : r0) + (lane & 15)), (lds_void*)&aux_s[wave][buf][(AUX - 1) * 64], 4, 0, 0);
    }
    // (every wave issues the same number of pieces: where there are fewer, some are fetched twice)
#pragma unroll
    for (int it = 0; it < KIT; ++it) {
      const int p = KP % NW == 0 ? wave + NW * it : (wave + NW * it) % KP;
      const int r0 = p * (64 / KCH), dr = lane / KCH, c = (lane % KCH) ^ (ONE ? kv_swz<DK>(r0 + dr) : k_swz<DK>(r0 + dr));
      __builtin_amdgcn_global_load_lds((glb_void*)(k_cache + (piece_row(kb + r0) + dr) * KST + c * 8), (lds_void*)(pf_lds + buf * KT + p * 512), 16, 0, 0);
    }
#pragma unroll
    for (int it = 0; it < VIT; ++it) {
      const int p = VP % NW == 0 ? wave + NW * it : (wave + NW * it) % (VP > 0 ? VP : 1);
      const int r0 = p * (64 / VCH), dr = lane / VCH, c = (lane % VCH) ^ (ONE ? kv_swz<D2>(r0 + dr) : v_swz<D2>(r0 + dr));
      __builtin_amdgcn_global_load_lds((glb_void*)((ONE ? k_cache + DK : v_cache) + (piece_row(kb + r0) + dr) * VST + c * 8), (lds_void*)(pf_lds + 3 * KT + buf * VT + p * 512), 16, 0, 0);
    }
  };

  // steps: the kept keys in front of the window, then the window
  const int kb0 = first & ~31;
  const int kept = (a.see.keep + 31) & ~31, kept_end = kept < kb0 ? kept : kb0;
  const int n_steps = (kept_end >> 5) + ((last - kb0) >> 5) + 1;
  auto step_key = [&](int i) { return 32 * i < kept_end ? 32 * i : kb0 + 32 * i - kept_end; };
  stage(step_key(0), 0);
  stage(step_key(1), 1);
  int buf = 0, ahead = 2;
  for (int i = 0; i < n_steps; ++i, buf = buf == 2 ? 0 : buf + 1, ahead = ahead == 2 ? 0 : ahead + 1) {
    asm volatile("s_waitcnt vmcnt(%0)" ::"n"(KIT + VIT + AUX) : "memory");  // (the youngest stage may still be on its way)
    __builtin_amdgcn_s_barrier();  // this step's rows have landed; every wave is done with the stage before
    const int kb = step_key(i);
    stage(step_key(i + 2), ahead);
    const bf16raw* k_img = pf_lds + buf * KT;
    const bf16raw* v_img = pf_lds + 3 * KT + buf * VT;
    if (!head_on) continue;
    const bool edge = kb + 31 > pos0 || kb < last_first || kb < first;
    frag_acc st = no_scores();
    if constexpr (RT > 0) {
      const bf16raw* r_img = v_img;
#pragma unroll
      for (int ks = 0; ks < RT / 16; ++ks)
        st = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const frag_ab*>(&r_img[lr * RT + (((2 * ks + hi) ^ kv_swz<RT>(lr)) << 3)]), qr[ks], st, 0, 0, 0);
    }
    const float* rs = &aux_s[wave][buf][0] + lr + 4 - 4 * hi;
    raw16 ks4[4] = {};  // the factors of register 4 g + e's key 8 g + 4 hi + e: on their way during the products (the compiler would wait for the LDS-DMA)
    if constexpr (ONE) {
      const unsigned int at = (unsigned int)(uintptr_t)(lds_void*)&aux_s[wave][buf][(AUX - 1) * 64 + 4 * hi];
      ks4[0] = lds_read16_at<0>(at); ks4[1] = lds_read16_at<32>(at); ks4[2] = lds_read16_at<64>(at); ks4[3] = lds_read16_at<96>(at);
    }
    attend_tile<DK, DV, ONE>(k_img, ONE ? k_img : v_img, qa, o, m_run, l_run, a.scale_log2e, edge, qpos - kb, q_first - kb, st, a.see.keep - kb, [&](int r, float v) __attribute__((always_inline)) {
      if constexpr (ONE) {
        if (r == 0) {  // (behind the factors' reads come the values' first ones, DV / 16 of them)
          asm volatile("s_waitcnt lgkmcnt(%4)" : "+v"(ks4[0]), "+v"(ks4[1]), "+v"(ks4[2]), "+v"(ks4[3]) : "n"(DV / 16 < 15 ? DV / 16 : 15));
        }
        v *= __uint_as_float(ks4[r >> 2][r & 3]);
      }
      if constexpr (REL) v += LOG2E * rs[27 - 8 * (r >> 2) - (r & 3)];
      return v;
    });
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // no piece may be in flight when the workgroup gives its LDS back
  const float l = l_run + __shfl_xor(l_run, 32, 64);
  if (!head_on || lr >= nq) return;
  float f = a.out_scale / l;
  const long long row = row0 + lr;
  if (a.gated == 1) f *= sigmoid(bf2f(gate[row * a.ld_gate + a.gate_off + head]));
  bf16raw* op = out + row * a.ldo + a.o_off + (long long)head * a.vdim;
  const bool vec = (a.vdim & 3) == 0 && (a.ldo & 3) == 0 && (a.o_off & 3) == 0 && (a.gated != 2 || ((a.ld_gate | a.gate_off) & 3) == 0);
  const bf16raw* gp = a.gated == 2 ? gate + row * a.ld_gate + a.gate_off + (long long)head * a.vdim : nullptr;
#pragma unroll
  for (int n = 0; n < DV / 32; ++n)
#pragma unroll
    for (int rr = 0; rr < 4; ++rr) {
      const int d = 32 * n + 8 * rr + 4 * hi;  // dims d .. d + 3 of this query
      float4 v = make_float4(o[n][4 * rr] * f, o[n][4 * rr + 1] * f, o[n][4 * rr + 2] * f, o[n][4 * rr + 3] * f);
      if (gp && d < a.vdim) {
        float4 z = make_float4(0.f, 0.f, 0.f, 0.f);
        if (vec) {
          z = ld4(gp + d);
        } else {
          z.x = ld(gp + d);
          if (d + 1 < a.vdim) z.y = ld(gp + d + 1);
          if (d + 2 < a.vdim) z.z = ld(gp + d + 2);
          if (d + 3 < a.vdim) z.w = ld(gp + d + 3);
        }
        v.x *= sigmoid(z.x); v.y *= sigmoid(z.y); v.z *= sigmoid(z.z); v.w *= sigmoid(z.w);
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

template <int DK, int DV, bool REL, int RT>
int launch_prefill(const void* q, const void* kc, const void* vc, const void* gate, void* out, int n_blocks, const ChunkAttnArgs& a, hipStream_t s) {
  const int rep = a.nh / a.nkv;
  constexpr size_t lds = (size_t)3 * 32 * (DK + (RT >= 0 ? RT : DV)) * sizeof(bf16raw);
#define KV_CP(NW)                                                                                                                                                          \
  if (lds > 65536 && hipFuncSetAttribute((const void*)chunk_prefill_kernel<DK, DV, NW, REL, RT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) return -1;     \
  hipLaunchKernelGGL((chunk_prefill_kernel<DK, DV, NW, REL, RT>), dim3(n_blocks, a.nkv, (rep + NW - 1) / NW), dim3(64 * NW), lds, s, (const bf16raw*)q, (const bf16raw*)kc, (const bf16raw*)vc, \
                     (const bf16raw*)gate, (bf16raw*)out, a)
  if (rep == 1) { KV_CP(1); }
  else if (rep == 2) { KV_CP(2); }
  else if (rep <= 4 || DV > 128) { KV_CP(4); }
  else {
    if constexpr (DV <= 128) { KV_CP(8); }  // (larger heads: eight waves leave too few registers)
  }
#undef KV_CP
  return (int)hipGetLastError();
}

// ---- decoding: one query per sequence -----------------------------------------------------------------------------
// grid (listed rows, key heads x groups of 16 query heads, shares): the keys a row sees, in blocks of 16 dealt out to the waves of its
// workgroups.  A wave multiplies a K block, straight from memory as the A operand, with the up to 16 query heads as columns
// (S^T: a lane owns one head and 4 keys), and the weights, already in the A layout of mfma_f32_16x16x16_bf16, with the V block, which
// passes through a piece of LDS of the wave's own for the transposed reads.  K / V of the next block are in flight meanwhile.
// FUSED: the kernel also does what norm_rope_write_kernel does for the row (query / key norm, rotation, K / V write).
// RT >= 0 (one row is key and value): the keys' operands come out of the piece of LDS, too.
// SPLIT: partial results (maximum, sum, unnormalised output per head) go to a workspace for chunk_decode_combine_kernel.
struct ChunkDecodeArgs {
  float* key_scale;  // RT >= 0: [cache rows]
  const int* block_tables; int max_blocks;
  const int* rows; const int* tok_seq; const int* positions; const int* slots;
  int nh, nkv, dim, vdim, bs_shift, shares;
  Sight see;
  float scale_log2e, out_scale, eps;
  long long ld_gate; int gate_off, gated;
  long long ldo; int o_off;
  // FUSED
  long long ldp; int q_off, k_off, v_off, rot_dims;
  const float* bias; const float* q_norm; const float* k_norm; const float* cos_t; const float* sin_t;
  float* part;  // SPLIT: [row][head][share][2 + DV]
};

template <int DK, int DV, int NW, bool FUSED, bool SPLIT, bool REL, int RT>
__global__ __launch_bounds__(64 * NW) void chunk_decode_kernel(const bf16raw* __restrict__ q, const bf16raw* __restrict__ proj, bf16raw* k_cache, bf16raw* v_cache,
                                                               const bf16raw* __restrict__ gate, bf16raw* __restrict__ out, ChunkDecodeArgs a) {
  constexpr int VCH = DV / 8, VIT = 16 * VCH / 64 > 0 ? 16 * VCH / 64 : 1;  // 16-byte pieces of a V row; of a V block per lane
  constexpr bool ONE = RT >= 0;
  constexpr int RW = ONE ? RT : 0, KST = DK + RW, VST = ONE ? KST : DV;  // row strides in the cache
  constexpr int QS = KST + 8;
  __shared__ __attribute__((aligned(16))) bf16raw q_s[16 * QS];
  __shared__ __attribute__((aligned(16))) unsigned char work[NW * 16 * DV * 4];  // per wave: a V block, later its output
  __shared__ float ml[NW][16][2];
  const int t = a.rows[blockIdx.x];
  if (t < 0 || a.slots[t] < 0) return;  // unused entry, or a padding row: it has no place in the cache
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63;
  const int lr = lane & 15, lq = lane >> 4;
  const int rep = a.nh / a.nkv, groups = (rep + 15) / 16;
  const int g = blockIdx.y / groups, h0 = (blockIdx.y % groups) * 16;  // key head, first query head inside its group
  const int nhd = rep - h0 < 16 ? rep - h0 : 16;
  const int pos = a.positions[t];
  const int first = first_seen(a.see, pos);
  const int b0 = first >> 4, kept = (a.see.keep + 15) >> 4, nk = kept < b0 ? kept : b0;
  const int nb = nk + (pos >> 4) - b0 + 1;  // blocks of 16 keys: kept ones in front of the window, then the window
  auto block_key = [&](int b) { return (b < nk ? b : b0 + b - nk) << 4; };
  const int stride = a.shares * NW;
  const int me = blockIdx.z * NW + wave;
  const int* __restrict__ bt = a.block_tables + (long long)a.tok_seq[t] * a.max_blocks;
  const int bs_mask = (1 << a.bs_shift) - 1;

  if constexpr (FUSED) {
    const bool owner = (nb - 1) % stride / NW == (int)blockIdx.z;  // this workgroup reads the block with the new key
    float* w = reinterpret_cast<float*>(work) + wave * DK;
    const bf16raw* pr = proj + (long long)t * a.ldp;
    const int half = a.rot_dims >> 1;
    const int slot = a.slots[t];
    const long long crow = ((long long)(slot >> a.bs_shift) * a.nkv + g) * (bs_mask + 1) + (slot & bs_mask);
    const int n_units = owner ? (ONE ? nhd + 1 : nhd + 2) : nhd;  // (more than 16 heads: every group's workgroup writes the same key)
    for (int u = wave; u < n_units; u += NW) {
      if (!ONE && u == nhd + 1) {  // value
        for (int i = lane; i < DV; i += 64)
          v_cache[crow * DV + i] = i < a.vdim ? f2bf(bf2f(pr[a.v_off + g * a.vdim + i]) + a.bias[(a.nh + a.nkv) * a.dim + g * a.vdim + i]) : (bf16raw)0;
        continue;
      }
      const bool is_q = u < nhd;
      const int hd = is_q ? g * rep + h0 + u : g;
      const bf16raw* src = pr + (is_q ? a.q_off : a.k_off) + hd * a.dim;
      const float* bias = a.bias + (is_q ? hd : a.nh + hd) * a.dim;
      const float* nw = is_q ? a.q_norm : a.k_norm;
      float x[DK / 64], ss = 0.f;
#pragma unroll
      for (int e = 0; e < DK / 64; ++e) {
        const int i = lane + 64 * e;
        x[e] = i < a.dim ? bf2f(src[i]) + bias[i] : 0.f;
        ss += x[e] * x[e];
      }
      const float rs = 1.f / sqrtf(wave_sum(ss) / (float)a.dim + a.eps);
#pragma unroll
      for (int e = 0; e < DK / 64; ++e) {
        const int i = lane + 64 * e;
        if constexpr (ONE) w[i] = i < a.dim ? (is_q ? x[e] * rs * nw[i] : x[e] * nw[i]) : 0.f;
        else w[i] = i < a.dim ? x[e] * rs * nw[i] : 0.f;
      }
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
#pragma unroll
      for (int e = 0; e < DK / 64; ++e) {
        const int i = lane + 64 * e;
        float v = w[i];
        if (i < a.rot_dims) {
          const int p = i < half ? i : i - half;
          const float c = a.cos_t[(long long)pos * half + p], s = a.sin_t[(long long)pos * half + p];
          v = i < half ? w[i] * c - w[i + half] * s : w[i] * c + w[i - half] * s;
        }
        if constexpr (ONE) {
          if (is_q) q_s[u * QS + i] = i < a.dim && i >= a.rot_dims ? f2bf(v * a.k_norm[i]) : (bf16raw)0;
          else k_cache[crow * KST + i] = f2bf(x[e]);
          if (i < RW) {
            const bf16raw z = i < a.rot_dims ? f2bf(v) : (bf16raw)0;
            if (is_q) q_s[u * QS + DK + i] = z;
            else k_cache[crow * KST + DK + i] = z;
          }
          if (!is_q && i == 0) a.key_scale[crow] = rs;
        } else {
          if (is_q) q_s[u * QS + i] = f2bf(v);
          else k_cache[crow * DK + i] = f2bf(v);
        }
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();
    }
    for (int i = tid; i < (16 - nhd) * KST; i += 64 * NW) q_s[(nhd + i / KST) * QS + i % KST] = 0;
    __threadfence_block();
  } else {
    for (int i = tid; i < 16 * (KST / 8); i += 64 * NW) {
      const int h = i / (KST / 8), c = i % (KST / 8);
      raw16 v = {0, 0, 0, 0};
      if (h < nhd) v = *reinterpret_cast<const raw16*>(q + ((long long)t * a.nh + g * rep + h0 + h) * KST + c * 8);
      *reinterpret_cast<raw16*>(&q_s[h * QS + c * 8]) = v;
    }
  }
  __syncthreads();
  frag_ab qb[KST / 32];
#pragma unroll
  for (int ks = 0; ks < KST / 32; ++ks) qb[ks] = *reinterpret_cast<const frag_ab*>(&q_s[lr * QS + ks * 32 + lq * 8]);
  __syncthreads();  // (FUSED: the scratch in `work` is free from here on)

  bf16raw* vl = reinterpret_cast<bf16raw*>(work) + wave * 32 * DV;
  frag_acc4 o[DV / 16];
#pragma unroll
  for (int n = 0; n < DV / 16; ++n) o[n] = (frag_acc4){0.f, 0.f, 0.f, 0.f};
  float m_run = -1e30f, l_run = 0.f;
  const int head_lr = g * rep + h0 + (lr < nhd ? lr : nhd - 1);  // the lane's head
  if (a.see.sink && me == 0) {  // (once per row)
    m_run = a.see.sink[head_lr] * LOG2E;
    l_run = lq == 0 ? 1.f : 0.f;
  }
  const float* rel = REL ? a.see.rel + (long long)head_lr * a.see.rel_n : nullptr;
  float rn[4] = {0.f, 0.f, 0.f, 0.f};
  constexpr int KF = ONE ? (RW > 0 ? RW / 32 : 1) : DK / 32;  // key operands straight from memory: all, or the rotated parts'
  raw16 kn[KF], vn[VIT];
  float4 sn = make_float4(1.f, 1.f, 1.f, 1.f);
  const int v_row = lane / VCH, v_c = lane % VCH;  // piece `it` of a V block: row v_row + it * (64 / VCH)
  auto fetch = [&](int b) __attribute__((always_inline)) {
    const int key = block_key(b);
    if constexpr (REL) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        int d = pos - key - 4 * lq - r;
        d = d < 0 ? 0 : d;
        rn[r] = rel[d < a.see.rel_n ? d : a.see.rel_n - 1];
      }
    }
    const long long page = ((long long)bt[key >> a.bs_shift] * a.nkv + g) * (bs_mask + 1) + (key & bs_mask);
    if constexpr (!ONE || RW > 0) {
      const bf16raw* kp = k_cache + (page + lr) * KST + (ONE ? DK : 0) + lq * 8;
#pragma unroll
      for (int ks = 0; ks < KF; ++ks) kn[ks] = *reinterpret_cast<const raw16*>(kp + ks * 32);
    }
    if constexpr (ONE) sn = ld4(a.key_scale + page + 4 * lq);
    const bf16raw* vp = ONE ? k_cache : v_cache;
#pragma unroll
    for (int it = 0; it < VIT; ++it) vn[it] = *reinterpret_cast<const raw16*>(vp + (page + v_row + it * (64 / VCH)) * VST + v_c * 8);
  };
  if (me < nb) fetch(me);
  for (int b = me; b < nb; b += stride) {
    raw16 kc[KF];
#pragma unroll
    for (int ks = 0; ks < KF; ++ks) kc[ks] = kn[ks];
    const float sk[4] = {sn.x, sn.y, sn.z, sn.w};
#pragma unroll
    for (int it = 0; it < VIT; ++it) {
      const int r = v_row + it * (64 / VCH);
      *reinterpret_cast<raw16*>(&vl[r * DV + ((v_c ^ (ONE ? kv_swz<DV>(r) : v_swz<DV>(r))) << 3)]) = vn[it];
    }
    float rc[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) rc[r] = rn[r];
    if (b + stride < nb) fetch(b + stride);
    frag_acc4 st = {0.f, 0.f, 0.f, 0.f};
    if constexpr (ONE) {
      if constexpr (RW > 0) {
#pragma unroll
        for (int ks = 0; ks < KF; ++ks) st = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(frag_ab, kc[ks]), qb[DK / 32 + ks], st, 0, 0, 0);
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");  // (the wave's rows are in its LDS)
#pragma unroll
      for (int ks = 0; ks < DK / 32; ++ks)
        st = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const frag_ab*>(&vl[lr * DV + (((4 * ks + lq) ^ kv_swz<DV>(lr)) << 3)]), qb[ks], st, 0, 0, 0);
    } else {
#pragma unroll
      for (int ks = 0; ks < KF; ++ks) st = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(frag_ab, kc[ks]), qb[ks], st, 0, 0, 0);
    }
    const int k0 = block_key(b) + 4 * lq;
    float sc[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      float v = st[r] * a.scale_log2e;
      if constexpr (ONE) v *= sk[r];
      if constexpr (REL) v += rc[r] * LOG2E;
      sc[r] = ((k0 + r >= first || k0 + r < a.see.keep) && k0 + r <= pos) ? v : -1e30f;
    }
    float mx = fmaxf(fmaxf(sc[0], sc[1]), fmaxf(sc[2], sc[3]));
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float m_new = fmaxf(m_run, mx);  // (a block holds at least one visible key)
    const float corr = __builtin_amdgcn_exp2f(m_run - m_new);
    typedef __attribute__((ext_vector_type(4))) __bf16 bf4;
    bf4 pb;
    float psum = 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float p = __builtin_amdgcn_exp2f(sc[r] - m_new);
      psum += p;
      pb[r] = (__bf16)p;
    }
    l_run = l_run * corr + psum;
    if (__builtin_amdgcn_ballot_w64(m_new != m_run) != 0) {
      float cr[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) cr[r] = __shfl(corr, 4 * lq + r, 64);  // output rows are heads 4 lq + r
#pragma unroll
      for (int n = 0; n < DV / 16; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[n][r] *= cr[r];
    }
    m_run = m_new;
    const frag_b64 pa = __builtin_bit_cast(frag_b64, pb);
#pragma unroll
    for (int n = 0; n < DV / 16; ++n) {
      const int r = 4 * lq + (lr >> 2), c = 2 * n + ((lr & 3) >> 1);
      const tr_b64 vf = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_tr_b64*)(&vl[r * DV + ((c ^ (ONE ? kv_swz<DV>(r) : v_swz<DV>(r))) << 3) + (lr & 1) * 4]));
      o[n] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(pa, __builtin_bit_cast(frag_b64, vf), o[n], 0, 0, 0);
    }
  }
  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  if (lq == 0) { ml[wave][lr][0] = m_run; ml[wave][lr][1] = l_run; }
  float* os = reinterpret_cast<float*>(work) + wave * 16 * DV;  // (the wave's own LDS: its reads above are done)
#pragma unroll
  for (int r = 0; r < 4; ++r)
    if (4 * lq + r < nhd) {
#pragma unroll
      for (int n = 0; n < DV / 16; ++n) os[(4 * lq + r) * DV + 16 * n + lr] = o[n][r];
    }
  __syncthreads();
  const float* oa = reinterpret_cast<const float*>(work);
  for (int i = tid; i < nhd * DV; i += 64 * NW) {
    const int h = i / DV, d = i % DV;
    if (d >= a.vdim) continue;
    float m = ml[0][h][0];
#pragma unroll
    for (int w = 1; w < NW; ++w) m = fmaxf(m, ml[w][h][0]);
    float l = 0.f, v = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      const float c = __builtin_amdgcn_exp2f(ml[w][h][0] - m);
      l += c * ml[w][h][1];
      v += c * oa[(w * 16 + h) * DV + d];
    }
    const int head = g * rep + h0 + h;
    if constexpr (SPLIT) {
      float* p = a.part + (((long long)blockIdx.x * a.nh + head) * a.shares + blockIdx.z) * (2 + DV);
      p[2 + d] = v;
      if (d == 0) { p[0] = m; p[1] = l; }
    } else {
      float f = a.out_scale / l;
      if (a.gated) f *= sigmoid(bf2f(gate[(long long)t * a.ld_gate + a.gate_off + (a.gated == 2 ? head * a.vdim + d : head)]));
      st(out + (long long)t * a.ldo + a.o_off + head * a.vdim + d, v * f);
    }
  }
}

template <int DV>
__global__ __launch_bounds__(64) void chunk_decode_combine_kernel(const bf16raw* __restrict__ gate, bf16raw* __restrict__ out, ChunkDecodeArgs a) {
  const int t = a.rows[blockIdx.x], head = blockIdx.y;
  if (t < 0 || a.slots[t] < 0) return;
  const float* p = a.part + ((long long)blockIdx.x * a.nh + head) * a.shares * (2 + DV);
  float m = -1e30f;
  for (int s = 0; s < a.shares; ++s) m = fmaxf(m, p[(long long)s * (2 + DV)]);
  float l = 0.f;
  for (int s = 0; s < a.shares; ++s) l += __builtin_amdgcn_exp2f(p[(long long)s * (2 + DV)] - m) * p[(long long)s * (2 + DV) + 1];
  float f = a.out_scale / l;
  if (a.gated == 1) f *= sigmoid(bf2f(gate[(long long)t * a.ld_gate + a.gate_off + head]));
  for (int d = threadIdx.x; d < a.vdim; d += 64) {
    float v = 0.f;
    for (int s = 0; s < a.shares; ++s) v += __builtin_amdgcn_exp2f(p[(long long)s * (2 + DV)] - m) * p[(long long)s * (2 + DV) + 2 + d];
    if (a.gated == 2) v *= sigmoid(bf2f(gate[(long long)t * a.ld_gate + a.gate_off + head * a.vdim + d]));
    st(out + (long long)t * a.ldo + a.o_off + head * a.vdim + d, v * f);
  }
}

template <int DK, int DV, bool REL, int RT>
int launch_decode(const void* q, const void* proj, void* kc, void* vc, const void* gate, void* out, int n_rows, bool fused, int waves, const ChunkDecodeArgs& a, hipStream_t s) {
  const int rep = a.nh / a.nkv;
  const dim3 grid(n_rows, a.nkv * ((rep + 15) / 16), a.shares);
#define KV_CD(NW, F, S) \
  hipLaunchKernelGGL((chunk_decode_kernel<DK, DV, NW, F, S, REL, RT>), grid, dim3(64 * NW), 0, s, (const bf16raw*)q, (const bf16raw*)proj, (bf16raw*)kc, (bf16raw*)vc, (const bf16raw*)gate, (bf16raw*)out, a)
#define KV_CD2(NW)                                                                  \
  do {                                                                              \
    if (a.shares > 1) { if (fused) KV_CD(NW, true, true); else KV_CD(NW, false, true); } \
    else { if (fused) KV_CD(NW, true, false); else KV_CD(NW, false, false); }       \
  } while (0)
  bool done = false;
  if constexpr (DV <= 128) {
    if (waves == 8) { KV_CD2(8); done = true; }
  }
  if (!done) KV_CD2(4);
#undef KV_CD2
#undef KV_CD
  if (a.shares > 1) hipLaunchKernelGGL((chunk_decode_combine_kernel<DV>), dim3(n_rows, a.nh), dim3(64), 0, s, (const bf16raw*)gate, (bf16raw*)out, a);
  return (int)hipGetLastError();
}

}  // namespace

extern "C" {

int kvc_supported(int dkp, int dvp);
int kvc_one_supported(int dvp, int rt, int rel);

// rows: listed token rows (-1 = unused); proj != nullptr: fused form (q unused).  key_scale != nullptr: one row is key and value (k_cache, rows of
// dvp and rt elements; dkp = dvp, v_cache unused)
int kvc_decode(const void* q, const void* proj, long long ldp, int q_off, int k_off, int v_off, const float* bias, const float* q_norm, const float* k_norm, const float* cos_t,
               const float* sin_t, int rot_dims, float eps, void* k_cache, void* v_cache, const int* block_tables, int max_blocks, const int* rows, int n_rows, const int* tok_seq,
               const int* positions, const int* slots, const void* gate, long long ld_gate, int gate_off, void* out, long long ldo, int o_off, int nh, int nkv, int dim, int dkp, int vdim,
               int dvp, int block_size, int chunk, int window, int keep, int gated, const float* sink, const float* rel, int rel_n, float scale, float out_scale, int waves, int shares, float* part,
               float* key_scale, int rt, hipStream_t s) {
  if (n_rows <= 0 || nh <= 0 || nkv <= 0 || nh % nkv || !kvc_supported(dkp, dvp) || dim <= 0 || dim > dkp || vdim <= 0 || vdim > dvp || chunk < 0 || window < 0 || keep < 0 || (rel && rel_n < 1) || (gated && !gate) || block_size < 16 ||
      (block_size & (block_size - 1)) || shares < 1 || (shares > 1 && !part) || (!proj && !q) || rot_dims > dim || (rot_dims & 1) || (key_scale && (dkp != dvp || dim != vdim || rt < rot_dims || !kvc_one_supported(dvp, rt, rel != nullptr)))) return -1;
  int shift = 0;
  while ((1 << shift) < block_size) ++shift;
  const ChunkDecodeArgs a{key_scale, block_tables, max_blocks, rows, tok_seq, positions, slots, nh, nkv, dim, vdim, shift, shares, Sight{chunk, window, keep, sink, rel, rel_n}, scale * LOG2E, out_scale, eps,
                          ld_gate, gate_off, gated, ldo, o_off, ldp, q_off, k_off, v_off, rot_dims, bias, q_norm, k_norm, cos_t, sin_t, part};
#define KV_LD3(DK, DV, REL, RT) launch_decode<DK, DV, REL, RT>(q, proj, k_cache, v_cache, gate, out, n_rows, proj != nullptr, waves, a, s)
#define KV_LD2(DK, DV, REL) KV_LD3(DK, DV, REL, -1)
#define KV_LD(DK, DV) (rel ? KV_LD2(DK, DV, true) : KV_LD2(DK, DV, false))
#define KV_LD1(D) (rt == 0 ? (rel ? KV_LD3(D, D, true, 0) : KV_LD3(D, D, false, 0)) : rt == 32 ? KV_LD3(D, D, false, 32) : KV_LD3(D, D, false, 64))
  if (key_scale) return dvp == 64 ? KV_LD1(64) : dvp == 128 ? KV_LD1(128) : KV_LD1(256);
  if (dkp == 64) return dvp == 64 ? KV_LD(64, 64) : KV_LD(64, 128);
  if (dkp == 128) return dvp == 64 ? KV_LD(128, 64) : KV_LD(128, 128);
  return KV_LD(256, 256);
#undef KV_LD
#undef KV_LD1
#undef KV_LD2
#undef KV_LD3
}

// head sizes (padded, elements per cache row) the matrix-core kernels are built for
int kvc_supported(int dkp, int dvp) { return (dkp == 64 || dkp == 128) ? (dvp == 64 || dvp == 128) : (dkp == 256 && dvp == 256); }

// ... where one row is key and value: the values' padded size and the rotated part's; with a distance bias
int kvc_one_supported(int dvp, int rt, int rel) { return (dvp == 64 || dvp == 128 || dvp == 256) && (rt == 0 || (!rel && (rt == 32 || rt == 64))); }

int kvc_prefill(const void* q, const void* k_cache, const void* v_cache, const int* block_tables, int max_blocks, const int* blocks, int block_stride, int n_blocks, const void* gate, long long ld_gate,
                int gate_off, void* out, long long ldo, int o_off, int nh, int nkv, int dkp, int vdim, int dvp, int block_size, int chunk, int window, int keep, int gated, const float* sink,
                const float* rel, int rel_n, float scale, float out_scale, const float* key_scale, int rt, hipStream_t s) {
  if (n_blocks <= 0 || n_blocks > block_stride || nh <= 0 || nkv <= 0 || nh % nkv || !kvc_supported(dkp, dvp) || vdim <= 0 || vdim > dvp || chunk < 0 || window < 0 || keep < 0 || (rel && rel_n < 1) || (gated && !gate) || block_size <= 0 || (block_size & (block_size - 1)) ||
      (key_scale && (dkp != dvp || !kvc_one_supported(dvp, rt, rel != nullptr)))) return -1;
  int shift = 0;
  while ((1 << shift) < block_size) ++shift;
  const ChunkAttnArgs a{key_scale, block_tables, max_blocks, blocks, blocks + block_stride, blocks + 2 * block_stride, blocks + 3 * block_stride, nh, nkv, vdim, shift, Sight{chunk, window, keep, sink, rel, rel_n},
                        scale * LOG2E, out_scale, ld_gate, gate_off, gated, ldo, o_off};
#define KV_LP3(DK, DV, REL, RT) launch_prefill<DK, DV, REL, RT>(q, k_cache, v_cache, gate, out, n_blocks, a, s)
#define KV_LP(DK, DV) (rel ? KV_LP3(DK, DV, true, -1) : KV_LP3(DK, DV, false, -1))
#define KV_LP1(D) (rt == 0 ? (rel ? KV_LP3(D, D, true, 0) : KV_LP3(D, D, false, 0)) : rt == 32 ? KV_LP3(D, D, false, 32) : KV_LP3(D, D, false, 64))
  if (key_scale) return dvp == 64 ? KV_LP1(64) : dvp == 128 ? KV_LP1(128) : KV_LP1(256);
  if (dkp == 64) return dvp == 64 ? KV_LP(64, 64) : KV_LP(64, 128);
  if (dkp == 128) return dvp == 64 ? KV_LP(128, 64) : KV_LP(128, 128);
  return KV_LP(256, 256);
#undef KV_LP
#undef KV_LP1
#undef KV_LP3
}

}  // extern "C"
