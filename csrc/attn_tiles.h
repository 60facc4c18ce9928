// Pieces shared by the prompt attention kernels of gfx950 (chunk_attention.hip, latent_attention.hip): swizzled K / V images in
// LDS and one step of 32 keys against 32 queries per wave.
#pragma once
#include "elem.h"

namespace attn {
using namespace elem;

typedef __attribute__((ext_vector_type(8))) __bf16 frag_ab;
typedef __attribute__((ext_vector_type(16))) float frag_acc;
typedef __attribute__((ext_vector_type(4))) short tr_b64;
typedef __attribute__((address_space(3))) tr_b64 lds_tr_b64;
typedef __attribute__((address_space(3))) void lds_void;
typedef const __attribute__((address_space(1))) void glb_void;
typedef const __attribute__((address_space(4))) int scalar_int;
typedef __attribute__((ext_vector_type(4))) float frag_acc4;
typedef __attribute__((ext_vector_type(4))) short frag_b64;
typedef __attribute__((ext_vector_type(4))) unsigned int raw16;

// ds_read_b64_tr_b16 as inline assembly: in front of the builtin the compiler waits for every LDS-DMA in flight, also those of stages
// nobody reads yet.  The caller waits (lds_landed) before it uses the results.
__device__ inline tr_b64 lds_read_tr(const bf16raw* p) {
  tr_b64 v;
  const unsigned int addr = (unsigned int)(uintptr_t)(lds_void*)p;
  asm volatile("ds_read_b64_tr_b16 %0, %1" : "=v"(v) : "v"(addr));
  return v;
}
template <int N>
__device__ inline void lds_landed(tr_b64 (&v)[N]) {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
  for (int i = 0; i < N; ++i) asm volatile("" : "+v"(v[i]));  // (uses stay behind the wait)
}

// LDS reads at address + constant offset as inline assembly (the caller waits for them): 16 bytes, and the transposed 8 bytes
template <int OFF>
__device__ inline raw16 lds_read16_at(unsigned int addr) {
  raw16 v;
  asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(v) : "v"(addr), "n"(OFF));
  return v;
}
template <int OFF>
__device__ inline tr_b64 lds_read_tr_at(unsigned int addr) {
  tr_b64 v;
  asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(v) : "v"(addr), "n"(OFF));
  return v;
}

// swizzle of 16-byte pieces: rows of a 256-byte bank line, then the row index
template <int D> __device__ inline int k_swz(int row) { return D >= 128 ? row & 15 : (row >> 1) & 7; }
template <int D> __device__ inline int v_swz(int row) { return D >= 128 ? (row & 7) << 1 : ((row >> 1) & 3) << 1; }

// ... of an image that is read both ways, as keys and (transposed) as values; 32: a small one, read as keys
template <int D> __device__ inline int kv_swz(int row) {
  if (D >= 128) return ((row & 7) << 1) | ((row >> 3) & 1);
  return D == 64 ? (((row >> 1) & 3) << 1) | ((row >> 3) & 1) : (row >> 2) & 3;
}

__device__ __forceinline__ frag_acc no_scores() {
  frag_acc st;
#pragma unroll
  for (int r = 0; r < 16; ++r) st[r] = 0.f;
  return st;
}

// One step of 32 keys for a wave's 32 queries; k_img [32][DK], v_img [32][DV] swizzled by k_swz / v_swz.  S^T = K Q^T on
// mfma_f32_32x32x16_bf16 (A = keys, B = queries): a lane owns query lane & 31 and 16 of the keys; the exponentiated accumulators, packed to
// bf16, are the B operand of O^T += V^T P^T when the k dimension is read as the permutation slot(8 hi + j) = key 16 s + 8 (j / 4) + 4 hi +
// j % 4; V^T comes out of LDS by transposed 8-byte reads.  edge: the lane's query sees only the keys [first_key, last_key] of the step.
// st: what the scores start from (of key dimensions that are not in k_img).  Of the keys in front of first_key the lane's query also sees those
// in front of keep_key.  finish(r, score): what becomes of the scaled score of register r (key 8 (r / 4) + 4 hi + r % 4).
// ONE: k_img and v_img are the same image, swizzled by kv_swz.
struct AsItIs { __device__ __forceinline__ float operator()(int, float v) const { return v; } };
template <int DK, int DV, bool ONE = false, typename Finish = AsItIs>
__device__ __forceinline__ void attend_tile(const bf16raw* k_img, const bf16raw* v_img, const frag_ab (&qa)[DK / 16], frag_acc (&o)[DV / 32], float& m_run, float& l_run, float scale_log2e,
                                            bool edge, int last_key, int first_key, frag_acc st, int keep_key = 0, Finish finish = Finish()) {
  const int lane = threadIdx.x & 63, lr = lane & 31, hi = lane >> 5;
  const int vq = (lane >> 2) & 3, vp = lane & 3, vodd = (lane >> 4) & 1;
#pragma unroll
  for (int ks = 0; ks < DK / 16; ++ks) {
    const frag_ab kf = *reinterpret_cast<const frag_ab*>(&k_img[lr * DK + (((2 * ks + hi) ^ (ONE ? kv_swz<DK>(lr) : k_swz<DK>(lr))) << 3)]);
    st = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qa[ks], st, 0, 0, 0);
  }
  // V^T fragments of key half h, dims 32 n + lr: two transposed reads (4 keys each); the first half's are read under the softmax
  auto v_read = [&](int h, int n, int j) __attribute__((always_inline)) {
    const int r = 16 * h + 8 * j + 4 * hi + vq, c = 4 * n + 2 * vodd + (vp >> 1);
    return lds_read_tr(v_img + r * DV + ((c ^ (ONE ? kv_swz<DV>(r) : v_swz<DV>(r))) << 3) + (vp & 1) * 4);
  };
  tr_b64 v0[DV / 16], v1[DV / 16];
#pragma unroll
  for (int n = 0; n < DV / 32; ++n) {
    v0[2 * n] = v_read(0, n, 0);
    v0[2 * n + 1] = v_read(0, n, 1);
  }
  // accumulator register r: key 8 (r / 4) + 4 hi + r % 4
  float sc[16];
#pragma unroll
  for (int r = 0; r < 16; ++r) sc[r] = finish(r, st[r] * scale_log2e);
  if (edge) {
    const int hi_lim = last_key - 4 * hi, lo_lim = first_key - 4 * hi, keep_lim = keep_key - 4 * hi;
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int k = 8 * (r >> 2) + (r & 3);
      sc[r] = (k <= hi_lim && (k >= lo_lim || k < keep_lim)) ? sc[r] : -1e30f;
    }
  }
  float mx = sc[0];
#pragma unroll
  for (int r = 1; r < 16; ++r) mx = fmaxf(mx, sc[r]);
  mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
  const float m_old = m_run, m_new = fmaxf(m_old, mx);
  float psum = 0.f;
  frag_ab pb[2];
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    // (a query none of whose keys have come up yet: nothing counts)
    const float p = m_new > -1e29f ? __builtin_amdgcn_exp2f(sc[r] - m_new) : 0.f;
    psum += p;
    pb[r >> 3][r & 7] = (__bf16)p;
  }
  const float corr = __builtin_amdgcn_exp2f(m_old - m_new);
  l_run = l_run * corr + psum;
  m_run = m_new;
  if (__builtin_amdgcn_ballot_w64(m_new != m_old) != 0) {
#pragma unroll
    for (int n = 0; n < DV / 32; ++n)
#pragma unroll
      for (int r = 0; r < 16; ++r) o[n][r] *= corr;
  }
  lds_landed(v0);
#pragma unroll
  for (int n = 0; n < DV / 32; ++n) {
    v1[2 * n] = v_read(1, n, 0);
    v1[2 * n + 1] = v_read(1, n, 1);
  }
#pragma unroll
  for (int n = 0; n < DV / 32; ++n) {
    const struct { tr_b64 lo, hi; } vf = {v0[2 * n], v0[2 * n + 1]};
    o[n] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(frag_ab, vf), pb[0], o[n], 0, 0, 0);
  }
  lds_landed(v1);
#pragma unroll
  for (int n = 0; n < DV / 32; ++n) {
    const struct { tr_b64 lo, hi; } vf = {v1[2 * n], v1[2 * n + 1]};
    o[n] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(frag_ab, vf), pb[1], o[n], 0, 0, 0);
  }
}

}  // namespace attn
