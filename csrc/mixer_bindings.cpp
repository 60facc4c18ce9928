// Python bindings of the sequence-mixer kernels (csrc/mixer_kernels.hip, chunk_attention.hip, delta_rule.hip,
// latent_attention.hip, retention.hip, state_space.hip, experts.hip), part of the extension `kvmini._C`.  Shapes, types and devices are checked here before every launch; what a kernel indexes by values
// held on the device (slots, positions, block tables) is staged by the runner within the sizes checked here.

#include <torch/extension.h>
#include <c10/hip/HIPStream.h>
#include <hip/hip_runtime.h>

#include <algorithm>
#include <cmath>

struct KvdArgs {
  long long ldp, ldl;
  int q_off, k_off, v_off, b_off, z_off, gate_off;
  const float *conv_w, *a_log, *dt_bias, *o_norm;
  float* state;
  const int *tok_seq, *positions, *tok_kind, *tok_off;
  int heads, kv_heads, dim, vdim, taps, channels;
  float eps, out_scale;
  long long ldo; int o_off;
};

struct KvrArgs {
  long long ldp; int q_off, k_off, v_off, g_off;
  const float* log2_decay;
  const float* cos_t; const float* sin_t;
  int rot_dims, heads, dim, vdim, dimp, dvp;
  float k_scale, eps, out_scale;
  float* state;
  const int *tok_seq, *positions, *tok_kind;
  long long ldo; int o_off;
};

struct KvsArgs {
  long long ldp; int z_off, x_off, dt_off;
  const float *conv_w, *conv_b, *dt_bias, *a_log, *skip, *norm;
  int heads, groups, dim, vdim, dimp, dvp, taps, channels, norm_groups;
  float eps, out_scale;
  float* state;
  const int *tok_seq, *positions, *tok_kind, *tok_off;
  long long ldo; int o_off;
};

extern "C" {
int kvm_embed_stream(const void* table, int f32, const int* tokens, const int* feed, const long long* prev_ids, int n_prev, float* x, void* xb, float* keep, float scale,
                     const int* positions, const float* turns, int T, int H, int ld, int V, hipStream_t s);
int kvm_gated_residual(float* x, void* xb, int f32, const void* y, long long y_ld, long long y_stride, int y_slabs, const float* y_weights, const float* bias, const void* gate,
                       long long gate_ld, long long gate_stride, int gate_slabs, const float* gate_bias, const float* g, int g_step, const float* next_g, int next_step,
                       const float* join_rows, const float* join_vec, float mult, float eps, int T, int H, int ld, hipStream_t s);
int kvm_latent_write(const void* proj, int f32, long long ldp, int c_off, const float* gain, const int* slots, const int* positions, void* cache, int write, int T, int rank, int rkp, int rot, int rtp,
                     int kr_off, const float* cos_t, const float* sin_t, int nh, int r_off, void* dst, long long ldd, int d_off, int d_head, float eps, hipStream_t s);
int kvm_hyper_residual(float* x, int streams, void* xb, int f32, const void* y, long long y_ld, long long y_stride, int y_slabs, const float* y_weights, const void* y2, long long y2_ld,
                       long long y2_stride, int y2_slabs, const float* gate2, const float* mix, const float* out, const float* read, const float* next_g, const float* start, float eps, int T, int H,
                       int ld, hipStream_t s);
int kvm_parallel_residual(float* x, void* xb, void* xb2, int f32, const void* y, long long y_ld, long long y_stride, int y_slabs, const void* y2, long long y2_ld, int top, const float* y2_weights,
                          const void* y3, long long y3_ld, long long y3_stride, int y3_slabs, const float* bias, const float* g, const float* g2, float eps, int T, int H, int ld, hipStream_t s);
int kvs_step(const KvsArgs* a, const void* proj, void* ring, float* y, int f32, const int* rows, int n_rows, hipStream_t s);
long long kvs_workspace(const KvsArgs* a, int n_rows, int n_chunks);
int kvs_portions(const KvsArgs* a, const void* proj, void* ring, float* y, int f32, void* xbc, float* ws, int n_rows, const int* segs, int n_segs, const int* chunks, int chunk_stride, int n_chunks,
                 const int* first_chunk, hipStream_t s);
int kvs_gate(const KvsArgs* a, const void* proj, const float* y, void* out, int f32, int n_rows, hipStream_t s);
int kvm_softcap(void* x, int f32, long long stride, int S, int V, float cap, hipStream_t s);
int kvr_chunked(int vdim);
int kvr_rows(const KvrArgs* a, const void* proj, void* out, int f32, const int* rows, int n_rows, hipStream_t s);
int kvr_portions(const KvrArgs* a, const void* proj, void* out, int f32, const int* segs, int n_segs, const int* chunks, int chunk_stride, int n_chunks, const int* first_chunk, float* ws, hipStream_t s);
int kvm_head_rows(const void* x, int f32, long long ldx, int x_off, int x_head, const void* w, int nh, int N, int K, int n_true, const void* gate, long long ld_gate, int gate_off, int gate_each,
                  void* out, long long ldo, int o_off, int o_head, float out_scale, const int* slots, int T, hipStream_t s);
int kvl_supported(int dkp, int dvp, int rk);
int kvl_gather(const void* cache, void* ws, const int* first_row, const int* first_pos, const int* count, int n_seqs, const int* block_tables, int max_blocks, int block_size, int n_rows, int rk,
               hipStream_t s);
int kvl_prefill(const void* proj, long long ldp, int q_off, int r_off, int gate_off, int gate_each, const void* kv, long long ldkv, int v_off, const void* kr, long long ldkr, int rt, const int* blocks,
                int block_stride, int n_blocks, void* out, long long ldo, int o_off, int nh, int dkp, int vdim, int dvp, int window, float scale, float out_scale, hipStream_t s);
int kvl_absorb(const void* proj, long long ldp, int q_off, int c_off, const void* w, void* q_lat, void* cache, int write, const int* rows, int n_rows, const int* slots, const float* c_norm, int rank,
               float eps, int nh, int dkp, int rk, int rt, const int* positions, int r_off, int kr_off, int rot, int turn, const float* cos_t, const float* sin_t, hipStream_t s);
int kvl_decode(const void* q_lat, const void* cache, void* lat, float* part, const int* block_tables, int max_blocks, const int* rows, int n_rows, const int* tok_seq, const int* positions, const int* slots,
               int nh, int rk, int rt, int block_size, int window, float scale, int shares, hipStream_t s);
int kvl_up(const void* lat, const void* w, const void* proj, long long ldp, int gate_off, int gate_each, void* out, long long ldo, int o_off, const int* rows, int n_rows, const int* slots, int nh,
           int rk, int vdim, int dvp, float out_scale, int parts, hipStream_t s);
int kve_route(const void* h, int f32, long long ldh, const void* w, const float* correction, const int* slots, int T, int E, int Ep, int top, int K, int* expert_of, float* weight_of, int scores, float scale, float* shared_of, const float* bias,
              hipStream_t s);
int kve_group(const int* expert_of, int n_pairs, int E, int bm, int* order, int* tiles, int max_tiles, int* n_tiles, hipStream_t s);
int kve_rows(const void* w, const void* x, void* y, int f32, int mode, const int* expert_of, int n_pairs, int top, int E, int N, int K, long long ldx, long long ldy, float limit, float slope, float shift, hipStream_t s);
int kv_wide_gemm_grouped(const void* Wp, const void* x, void* out, int N, int K, long long ldx, long long ldy, int mode, float limit, float slope, float shift, int bm, int* order, int* tiles, int max_tiles, int* n_tiles,
                         int row_div, hipStream_t stream);
int kvm_norm_rope_write(const void* proj, int f32, void* q, void* k_cache, void* v_cache, long long ldp, int q_off, int k_off, int v_off, const float* bias, const float* q_norm,
                        const float* k_norm, const int* positions, const int* slots, const float* cos_t, const float* sin_t, int rot_dims, int T, int nh, int nkv, int dim, int vdim,
                        int dkp, int dvp, int block_size, float eps, hipStream_t s);
int kvm_row_attention(const void* q, int f32, const void* k_cache, const void* v_cache, const int* block_tables, int max_blocks, const int* tok_seq, const int* positions,
                      const int* slots, const void* gate, long long ld_gate, int gate_off, void* out, long long ldo, int o_off, int T, int nh, int nkv, int dkp, int vdim, int dvp,
                      int block_size, int chunk, int window, int keep, int gate_each, const float* sink, const float* rel, int rel_n, float scale, float out_scale, const int* row_flag, int only_flag,
                      hipStream_t s);
int kvm_argmax_f32(const float* logits, long long stride, int S, int V, long long* out, hipStream_t s);
int kvc_supported(int dkp, int dvp);
int kvc_prefill(const void* q, const void* k_cache, const void* v_cache, const int* block_tables, int max_blocks, const int* blocks, int block_stride, int n_blocks, const void* gate, long long ld_gate,
                int gate_off, void* out, long long ldo, int o_off, int nh, int nkv, int dkp, int vdim, int dvp, int block_size, int chunk, int window, int keep, int gated, const float* sink,
                const float* rel, int rel_n, float scale, float out_scale, const float* key_scale, int rt, hipStream_t s);
int kvc_one_supported(int dvp, int rt, int rel);
int kvm_key_value_write(const void* proj, void* q, void* cache, float* key_scale, int rt, long long ldp, int q_off, int k_off, const float* bias, const float* q_norm, const float* k_norm,
                        const int* positions, const int* slots, const float* cos_t, const float* sin_t, int rot_dims, int T, int nh, int nkv, int dim, int dvp, int block_size, float eps, hipStream_t s);
int kvd_step_rows(int dim, int vdim);
int kvc_decode(const void* q, const void* proj, long long ldp, int q_off, int k_off, int v_off, const float* bias, const float* q_norm, const float* k_norm, const float* cos_t,
               const float* sin_t, int rot_dims, float eps, void* k_cache, void* v_cache, const int* block_tables, int max_blocks, const int* rows, int n_rows, const int* tok_seq,
               const int* positions, const int* slots, const void* gate, long long ld_gate, int gate_off, void* out, long long ldo, int o_off, int nh, int nkv, int dim, int dkp, int vdim,
               int dvp, int block_size, int chunk, int window, int keep, int gated, const float* sink, const float* rel, int rel_n, float scale, float out_scale, int waves, int shares, float* part,
               float* key_scale, int rt, hipStream_t s);
int kvd_step(const KvdArgs* k, const void* proj, const void* low, void* ring, void* out, int f32, const int* row_list, int n_rows, hipStream_t s);
int kvd_tile_dkp(int dim);
long long kvd_tile_floats(int dkp, int dvp);
int kvd_tiles(const KvdArgs* k, const void* proj, const void* low, void* ring, int f32, const int* tiles, int tile_stride, int n_tiles, const int* segs, int n_segs, int min_n, float* ws,
              float* o, hipStream_t s);
int kvd_prep(const KvdArgs* k, const void* proj, const void* low, const void* ring, int f32, float* qn, float* kn, float* vv, float* dec, float* beta, int dimp, int min_kind, int T,
             hipStream_t s);
int kvd_scan(const float* qn, const float* kn, const float* vv, const float* dec, const float* beta, float* o, const int* segs, int n_segs, int min_n, int dimp, float* state, int heads,
             int kv_heads, int dim, int vdim, hipStream_t s);
int kvd_out(const KvdArgs* k, const float* o, const void* low, void* out, int f32, int min_kind, int T, hipStream_t s);
int kvd_conv_tail(const KvdArgs* k, const void* proj, void* ring, int f32, const int* segs, int n_segs, int min_n, hipStream_t s);
}

namespace {

using at::Tensor;
using OptT = c10::optional<Tensor>;

hipStream_t stream() {
  (void)hipGetLastError();  // (a stale error of an earlier call is not this launch's)
  return c10::hip::getCurrentHIPStream().stream();
}
void check(int rc, const char* what) { TORCH_CHECK(rc == 0, what, " failed (", rc, rc > 0 ? hipGetErrorString((hipError_t)rc) : ": shapes outside the kernel's range", ")"); }

bool is_f32(const Tensor& t) {
  TORCH_CHECK(t.is_cuda() && (t.scalar_type() == at::kFloat || t.scalar_type() == at::kBFloat16), "bf16 or fp32 GPU tensor expected");
  return t.scalar_type() == at::kFloat;
}
void rows2d(const Tensor& t, at::ScalarType ty, int64_t rows, int64_t cols, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == ty && t.dim() == 2 && t.size(0) >= rows && t.size(1) >= cols && t.stride(1) == 1, what, ": [", rows, ", ", cols, "] rows expected, got ", t.sizes());
}
const float* f32p(const OptT& t, int64_t n, const char* what) {
  if (!t.has_value()) return nullptr;
  TORCH_CHECK(t->is_cuda() && t->scalar_type() == at::kFloat && t->is_contiguous() && t->numel() >= n, what, " must be contiguous fp32 with at least ", n, " entries");
  return (const float*)t->data_ptr();
}
const int* i32p(const Tensor& t, int64_t n, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kInt && t.is_contiguous() && t.numel() >= n, what, " must be contiguous int32 with at least ", n, " entries");
  return (const int*)t.data_ptr();
}

// keep: a second copy of x; turns: fp32 [columns / 2 rounded up, 2], frequencies of the sines and cosines to add, in turns, as sums of two floats
void embed_stream(Tensor table, Tensor tokens, Tensor feed, Tensor prev_ids, Tensor x, Tensor xb, OptT keep, double scale, OptT positions, OptT turns) {
  const bool f = is_f32(table);
  const int64_t T = tokens.numel(), H = table.size(1);
  TORCH_CHECK(table.dim() == 2 && table.is_contiguous() && prev_ids.scalar_type() == at::kLong && prev_ids.is_contiguous() && prev_ids.is_cuda(), "embed_stream: bad table or previous ids");
  rows2d(x, at::kFloat, T, H, "stream");
  rows2d(xb, table.scalar_type(), T, H, "projection input");
  TORCH_CHECK(x.is_contiguous() && xb.is_contiguous() && x.size(1) == xb.size(1), "embed_stream: rows of one width");
  check(kvm_embed_stream(table.data_ptr(), f, i32p(tokens, T, "tokens"), i32p(feed, T, "feed"), (const long long*)prev_ids.data_ptr(), (int)prev_ids.numel(), (float*)x.data_ptr(), xb.data_ptr(),
                         (float*)f32p(keep, T * x.size(1), "copy of the stream"), (float)scale, turns.has_value() ? i32p(positions.value(), T, "positions") : nullptr,
                         f32p(turns, (H + 1) / 2 * 2, "frequencies"), (int)T, (int)H, (int)x.size(1), (int)table.size(0), stream()), "embed_stream");
}

// rows [T, >= ld] of type ty, or fp32 slabs [S, T, ld] to be summed
struct Rows { const void* p = nullptr; long long ld = 0, stride = 0; int n = 0; };
Rows row_source(const Tensor& t, at::ScalarType ty, int64_t T, int64_t ld, const char* what) {
  Rows r;
  TORCH_CHECK(t.is_cuda(), what, ": GPU tensors");
  if (t.dim() == 3) {
    TORCH_CHECK(t.scalar_type() == at::kFloat && t.stride(2) == 1 && t.size(1) >= T && t.size(2) >= ld, what, ": slabs [S, T, ld] fp32");
    r.ld = t.stride(1); r.stride = t.stride(0); r.n = (int)t.size(0);
  } else {
    rows2d(t, ty, T, ld, what);
    r.ld = t.stride(0);
  }
  TORCH_CHECK(((uintptr_t)t.data_ptr() % (4 * t.element_size())) == 0 && r.ld % 4 == 0, what, ": rows must be aligned to four elements");
  r.p = t.data_ptr();
  return r;
}

// y, gate: fp32 slabs [S, T, ld] or rows [T, >= ld] of xb's type; y also [T * n, >= ld] with y_weights [T, n], or None.  Gains: 1 or ld entries.
void gated_residual(Tensor x, Tensor xb, OptT y, OptT y_weights, OptT bias, OptT gate, OptT gate_bias, OptT g, OptT next_g, OptT join_rows, OptT join_vec, double mult, double eps, int64_t width) {
  const bool f = is_f32(xb);
  const int64_t T = x.size(0), ld = x.size(1);
  TORCH_CHECK(x.is_contiguous() && xb.is_contiguous() && xb.size(0) == T && xb.size(1) == ld && x.scalar_type() == at::kFloat && x.is_cuda(), "gated_residual: stream and projection input of one shape");
  TORCH_CHECK(width <= ld && ld % 4 == 0, "gated_residual: bad width");
  Rows ys, gs;
  if (y.has_value()) {
    TORCH_CHECK(g.has_value(), "gated_residual: a result needs its norm");
    ys = row_source(*y, xb.scalar_type(), T, ld, "gated_residual");
    if (y_weights.has_value()) {
      TORCH_CHECK(y_weights->dim() == 2 && y_weights->size(0) == T && y_weights->size(1) >= 1 && y->dim() == 2 && y->size(0) >= T * y_weights->size(1), "gated_residual: weighted rows [T n, ld], weights [T, n]");
      ys.n = (int)y_weights->size(1);
    }
  }
  auto step = [&](const OptT& t) {
    TORCH_CHECK(!t.has_value() || t->numel() == 1 || t->numel() >= ld, "gated_residual: one gain, or one per column");
    return t.has_value() && t->numel() > 1 ? 1 : 0;
  };
  if (gate.has_value()) {
    gs = row_source(*gate, xb.scalar_type(), T, ld, "gated_residual");
    TORCH_CHECK(gate_bias.has_value(), "gated_residual: a gate needs its bias");
  }
  check(kvm_gated_residual((float*)x.data_ptr(), xb.data_ptr(), f, ys.p, ys.ld, ys.stride, ys.n, f32p(y_weights, 1, "row weights"), f32p(bias, ld, "bias"), gs.p, gs.ld, gs.stride, gs.n,
                           f32p(gate_bias, ld, "gate bias"), f32p(g, 1, "norm"), step(g), f32p(next_g, 1, "next norm"), step(next_g), f32p(join_rows, T * ld, "joining rows"),
                           f32p(join_vec, ld, "joining vector"), (float)mult, (float)eps, (int)T, (int)width, (int)ld, stream()), "gated_residual");
}

// x: streams fp32 [T, n, ld].  y: fp32 slabs [S, T, ld], rows [T, >= ld] of xb's type, or weighted rows [T k, >= ld] with y_weights [T, k];
// y2 (slabs or rows) is added times gate2 [T].  mix [n, n] (from, to), out and read [n], next_g [ld].  start [T, ld]: the streams begin as it.
void hyper_residual(Tensor x, Tensor xb, OptT y, OptT y_weights, OptT y2, OptT gate2, OptT mix, OptT out, Tensor read, Tensor next_g, OptT start, double eps, int64_t width) {
  const bool f = is_f32(xb);
  TORCH_CHECK(x.dim() == 3 && x.is_contiguous() && x.is_cuda() && x.scalar_type() == at::kFloat && xb.is_contiguous() && xb.dim() == 2 && xb.size(0) == x.size(0) && xb.size(1) == x.size(2),
              "hyper_residual: streams fp32 [T, n, ld], rows [T, ld]");
  const int64_t T = x.size(0), n = x.size(1), ld = x.size(2);
  TORCH_CHECK(width <= ld && ld % 4 == 0 && read.numel() == n, "hyper_residual: bad width or weights");
  Rows ys, zs;
  if (y.has_value()) {
    ys = row_source(*y, xb.scalar_type(), T, ld, "hyper_residual");
    if (y_weights.has_value()) {
      TORCH_CHECK(y_weights->dim() == 2 && y_weights->size(0) == T && y_weights->size(1) >= 1 && y->dim() == 2 && y->size(0) >= T * y_weights->size(1), "hyper_residual: weighted rows [T k, ld], weights [T, k]");
      ys.n = (int)y_weights->size(1);
    }
  }
  if (y2.has_value()) zs = row_source(*y2, xb.scalar_type(), T, ld, "hyper_residual");
  check(kvm_hyper_residual((float*)x.data_ptr(), (int)n, xb.data_ptr(), f, ys.p, ys.ld, ys.stride, ys.n, f32p(y_weights, 1, "row weights"), zs.p, zs.ld, zs.stride, zs.n, f32p(gate2, T, "row gates"),
                           f32p(mix, n * n, "stream mix"), f32p(out, n, "stream outputs"), f32p(read, n, "stream inputs"), f32p(next_g, ld, "next norm"), f32p(start, T * ld, "start rows"), (float)eps,
                           (int)T, (int)width, (int)ld, stream()), "hyper_residual");
}

// y, y3: fp32 slabs [S, T, ld] or rows [T, >= ld] of xb's type; y2: rows [T n, >= ld] weighted by y2_weights [T, n]; xb2 with next_g2
void parallel_residual(Tensor x, Tensor xb, OptT xb2, OptT y, OptT y2, OptT y2_weights, OptT y3, OptT bias, Tensor next_g, OptT next_g2, double eps, int64_t width) {
  const bool f = is_f32(xb);
  const int64_t T = x.size(0), ld = x.size(1);
  auto like = [&](const Tensor& t) { return t.is_contiguous() && t.dim() == 2 && t.size(0) == T && t.size(1) == ld && t.scalar_type() == xb.scalar_type() && t.is_cuda(); };
  TORCH_CHECK(x.is_contiguous() && x.dim() == 2 && x.scalar_type() == at::kFloat && x.is_cuda() && like(xb) && (!next_g2.has_value() || (xb2.has_value() && like(*xb2))), "parallel_residual: stream and products' inputs of one shape");
  TORCH_CHECK(width <= ld && ld % 4 == 0, "parallel_residual: bad width");
  Rows a, b, c;
  int top = 0;
  if (y.has_value()) a = row_source(*y, xb.scalar_type(), T, ld, "parallel_residual");
  if (y2.has_value()) {
    TORCH_CHECK(y2->dim() == 2 && y2_weights.has_value() && y2_weights->dim() == 2 && y2_weights->size(0) == T && y2_weights->size(1) >= 1 && y2->size(0) >= T * y2_weights->size(1),
                "parallel_residual: weighted rows [T n, ld], weights [T, n]");
    b = row_source(*y2, xb.scalar_type(), T, ld, "parallel_residual");
    top = (int)y2_weights->size(1);
  }
  if (y3.has_value()) c = row_source(*y3, xb.scalar_type(), T, ld, "parallel_residual");
  check(kvm_parallel_residual((float*)x.data_ptr(), xb.data_ptr(), xb2.has_value() ? xb2->data_ptr() : nullptr, f, a.p, a.ld, a.stride, a.n, b.p, b.ld, top, f32p(y2_weights, 1, "row weights"), c.p, c.ld,
                              c.stride, c.n, f32p(bias, ld, "bias"), f32p(next_g, ld, "next norm"), f32p(next_g2, ld, "next norm"), (float)eps, (int)T, (int)width, (int)ld, stream()), "parallel_residual");
}

void softcap(Tensor logits, double cap) {
  const bool f = is_f32(logits);
  TORCH_CHECK(logits.dim() == 2 && logits.stride(1) == 1, "softcap: rows of logits");
  check(kvm_softcap(logits.data_ptr(), f, logits.stride(0), (int)logits.size(0), (int)logits.size(1), (float)cap, stream()), "softcap");
}

struct CacheDims { int64_t blocks, nkv, bs, dkp, dvp; };
CacheDims cache_dims(const Tensor& k, const Tensor& v, at::ScalarType ty) {
  TORCH_CHECK(k.is_cuda() && v.is_cuda() && k.scalar_type() == ty && v.scalar_type() == ty && k.dim() == 4 && v.dim() == 4 && k.is_contiguous() && v.is_contiguous() && k.size(0) == v.size(0) &&
              k.size(1) == v.size(1) && k.size(2) == v.size(2), "K / V cache: contiguous [blocks, kv heads, block size, dim] of the activations' type");
  return {k.size(0), k.size(1), k.size(2), k.size(3), v.size(3)};
}

void norm_rope_write(Tensor proj, int64_t q_off, int64_t k_off, int64_t v_off, OptT bias, OptT q_norm, OptT k_norm, Tensor positions, Tensor slots, Tensor cos_t, Tensor sin_t, int64_t rot_dims,
                     Tensor q, Tensor k_cache, Tensor v_cache, int64_t dim, int64_t vdim, double eps) {
  const bool f = is_f32(proj);
  const CacheDims c = cache_dims(k_cache, v_cache, proj.scalar_type());
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous() && q.is_cuda() && q.scalar_type() == proj.scalar_type() && q.size(2) == c.dkp, "q must be contiguous [T, heads, padded dim]");
  const int64_t T = q.size(0), nh = q.size(1);
  rows2d(proj, proj.scalar_type(), T, std::max({q_off + nh * dim, k_off + c.nkv * dim, v_off + c.nkv * vdim}), "projections");
  TORCH_CHECK(rot_dims == 0 || (cos_t.dim() == 2 && cos_t.size(1) * 2 == rot_dims && cos_t.sizes() == sin_t.sizes()), "rotation tables must be [positions, rot_dims / 2]");
  check(kvm_norm_rope_write(proj.data_ptr(), f, q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), proj.stride(0), (int)q_off, (int)k_off, (int)v_off,
                            f32p(bias, nh * dim + c.nkv * (dim + vdim), "bias"), f32p(q_norm, dim, "query norm"), f32p(k_norm, dim, "key norm"), i32p(positions, T, "positions"),
                            i32p(slots, T, "slots"), f32p(cos_t, 0, "cos"), f32p(sin_t, 0, "sin"), (int)rot_dims, (int)T, (int)nh, (int)c.nkv, (int)dim, (int)vdim, (int)c.dkp, (int)c.dvp,
                            (int)c.bs, (float)eps, stream()), "norm_rope_write");
}

// sink [heads], rel [heads, distances]
struct Extra { const float* sink = nullptr; const float* rel = nullptr; int rel_n = 0; };
Extra extra(const OptT& sink, const OptT& rel, int64_t heads) {
  Extra e;
  e.sink = f32p(sink, heads, "sinks");
  if (rel.has_value()) {
    TORCH_CHECK(rel->dim() == 2 && rel->size(0) == heads && rel->size(1) >= 1, "distance biases [heads, distances]");
    e.rel = f32p(rel, heads, "distance biases");
    e.rel_n = (int)rel->size(1);
  }
  return e;
}
// gates: 0 none, 1 per head, 2 per element
int64_t gate_columns(int64_t gates, int64_t heads, int64_t vdim) {
  TORCH_CHECK(gates >= 0 && gates <= 2, "gates: 0 none, 1 per head, 2 per element");
  return gates == 2 ? heads * vdim : gates * heads;
}

// Where one row is key and value: v_cache is the fp32 factors that norm the keys, [blocks, kv heads, block size, 1], and a cache row has the
// rotated part behind the value.
struct OneRow { float* scale = nullptr; int64_t rt = 0; };
CacheDims one_row_dims(const Tensor& k, const Tensor& v, const Tensor& like, int64_t vdim, OneRow& one) {
  if (!(v.scalar_type() == at::kFloat && like.scalar_type() == at::kBFloat16)) return cache_dims(k, v, like.scalar_type());
  TORCH_CHECK(k.is_cuda() && v.is_cuda() && k.scalar_type() == at::kBFloat16 && k.dim() == 4 && v.dim() == 4 && k.is_contiguous() && v.is_contiguous() && k.size(0) == v.size(0) && k.size(1) == v.size(1) &&
              k.size(2) == v.size(2) && v.size(3) == 1, "rows [blocks, kv heads, block size, dim + rotated part], factors fp32 [blocks, kv heads, block size, 1]");
  const int64_t dvp = vdim <= 64 ? 64 : vdim <= 128 ? 128 : 256;
  one.scale = (float*)v.data_ptr();
  one.rt = k.size(3) - dvp;
  TORCH_CHECK(one.rt >= 0 && kvc_one_supported((int)dvp, (int)one.rt, 0), "rows of keys that are values: unsupported sizes");
  return {k.size(0), k.size(1), k.size(2), dvp, dvp};
}

// Queries and cache rows as the kernels take them where the values are the keys as projected
void key_value_write(Tensor proj, int64_t q_off, int64_t k_off, Tensor bias, Tensor q_norm, Tensor k_norm, Tensor positions, Tensor slots, Tensor cos_t, Tensor sin_t, int64_t rot_dims, Tensor q, Tensor rows,
                     Tensor scales, int64_t dim, double eps) {
  OneRow one;
  const CacheDims c = one_row_dims(rows, scales, proj, dim, one);
  TORCH_CHECK(one.scale && !is_f32(proj) && q.dim() == 3 && q.is_contiguous() && q.is_cuda() && q.scalar_type() == proj.scalar_type() && q.size(2) == rows.size(3), "q must be contiguous [T, heads, row]");
  const int64_t T = q.size(0), nh = q.size(1);
  rows2d(proj, proj.scalar_type(), T, std::max(q_off + nh * dim, k_off + c.nkv * dim), "projections");
  TORCH_CHECK(rot_dims == 0 || (cos_t.dim() == 2 && cos_t.size(1) * 2 == rot_dims && cos_t.sizes() == sin_t.sizes()), "rotation tables must be [positions, rot_dims / 2]");
  check(kvm_key_value_write(proj.data_ptr(), q.data_ptr(), rows.data_ptr(), one.scale, (int)one.rt, proj.stride(0), (int)q_off, (int)k_off, f32p(bias, (nh + c.nkv) * dim, "bias"), f32p(q_norm, dim, "query norm"),
                            f32p(k_norm, dim, "key norm"), i32p(positions, T, "positions"), i32p(slots, T, "slots"), f32p(cos_t, 0, "cos"), f32p(sin_t, 0, "sin"), (int)rot_dims, (int)T, (int)nh, (int)c.nkv,
                            (int)dim, (int)c.dvp, (int)c.bs, (float)eps, stream()), "key_value_write");
}

struct GateSrc { const void* p = nullptr; long long ld = 0; };
GateSrc gate_src(const OptT& gate, int64_t gate_off, const Tensor& q, int64_t nh) {
  if (!gate.has_value()) return {};
  rows2d(*gate, q.scalar_type(), q.size(0), gate_off + nh, "gates");
  return {gate->data_ptr(), gate->stride(0)};
}

void row_attention(Tensor q, Tensor k_cache, Tensor v_cache, Tensor block_tables, Tensor tok_seq, Tensor positions, Tensor slots, OptT gate, int64_t gate_off, int64_t gates, Tensor out, int64_t o_off, int64_t vdim,
                   int64_t chunk, int64_t window, int64_t keep, OptT sink, OptT rel, double scale, double out_scale, OptT row_flag, int64_t only_flag) {
  const bool f = is_f32(q);
  const CacheDims c = cache_dims(k_cache, v_cache, q.scalar_type());
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous() && q.size(2) == c.dkp, "q must be contiguous [T, heads, padded dim]");
  const int64_t T = q.size(0), nh = q.size(1);
  rows2d(out, q.scalar_type(), T, o_off + nh * vdim, "output");
  TORCH_CHECK(block_tables.dim() == 2, "block tables [sequences, blocks]");
  const GateSrc gs = gates ? gate_src(gate, gate_off, q, gate_columns(gates, nh, vdim)) : GateSrc{};
  TORCH_CHECK(!gates || gs.p, "row_attention: no gates");
  const Extra ex = extra(sink, rel, nh);
  check(kvm_row_attention(q.data_ptr(), f, k_cache.data_ptr(), v_cache.data_ptr(), i32p(block_tables, 1, "block tables"), (int)block_tables.size(1), i32p(tok_seq, T, "tok_seq"),
                          i32p(positions, T, "positions"), i32p(slots, T, "slots"), gs.p, gs.ld, (int)gate_off, out.data_ptr(), out.stride(0), (int)o_off, (int)T, (int)nh, (int)c.nkv, (int)c.dkp,
                          (int)vdim, (int)c.dvp, (int)c.bs, (int)chunk, (int)window, (int)keep, gates == 2, ex.sink, ex.rel, ex.rel_n, (float)scale, (float)out_scale, row_flag.has_value() ? i32p(*row_flag, T, "row flags") : nullptr, (int)only_flag, stream()),
        "row_attention");
}

// blocks: int32 [4, m]: first row, queries (0 = unused, at most 32), first position, block-table row; the first n_blocks in use at most
void chunk_prefill(Tensor q, Tensor k_cache, Tensor v_cache, Tensor block_tables, Tensor blocks, int64_t n_blocks, OptT gate, int64_t gate_off, int64_t gates, Tensor out, int64_t o_off, int64_t vdim, int64_t chunk,
                   int64_t window, int64_t keep, OptT sink, OptT rel, double scale, double out_scale) {
  TORCH_CHECK(!is_f32(q), "chunk_prefill: bf16");
  OneRow one;
  const CacheDims c = one_row_dims(k_cache, v_cache, q, vdim, one);
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous() && q.size(2) == c.dkp + one.rt, "q must be contiguous [T, heads, padded dim]");
  const int64_t T = q.size(0), nh = q.size(1);
  rows2d(out, q.scalar_type(), T, o_off + nh * vdim, "output");
  TORCH_CHECK(block_tables.dim() == 2 && blocks.dim() == 2 && blocks.size(0) == 4, "block tables [sequences, blocks], query blocks [4, n]");
  const GateSrc gs = gates ? gate_src(gate, gate_off, q, gate_columns(gates, nh, vdim)) : GateSrc{};
  const Extra ex = extra(sink, rel, nh);
  check(kvc_prefill(q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), i32p(block_tables, 1, "block tables"), (int)block_tables.size(1), i32p(blocks, 4, "query blocks"), (int)blocks.size(1), (int)n_blocks, gs.p,
                    gs.ld, (int)gate_off, out.data_ptr(), out.stride(0), (int)o_off, (int)nh, (int)c.nkv, (int)c.dkp, (int)vdim, (int)c.dvp, (int)c.bs, (int)chunk, (int)window, (int)keep, (int)gates, ex.sink, ex.rel,
                    ex.rel_n, (float)scale, (float)out_scale, one.scale, (int)one.rt, stream()), "chunk_prefill");
}

// Rows listed in `rows` (-1 = unused), one query each.  q [T, heads, padded dim] rotated, its keys in the cache; or q = None: query / key
// norm, rotation and the K / V write happen here, from the projections (columns q_off, k_off, v_off).
void chunk_decode(OptT q, Tensor proj, int64_t q_off, int64_t k_off, int64_t v_off, Tensor bias, Tensor q_norm, Tensor k_norm, Tensor cos_t, Tensor sin_t, int64_t rot_dims, double eps,
                  Tensor k_cache, Tensor v_cache, Tensor block_tables, Tensor rows, Tensor tok_seq, Tensor positions, Tensor slots, int64_t gate_off, int64_t gates, Tensor out, int64_t o_off, int64_t nh,
                  int64_t dim, int64_t vdim, int64_t chunk, int64_t window, int64_t keep, OptT sink, OptT rel, double scale, double out_scale, int64_t waves, int64_t shares) {
  TORCH_CHECK(!is_f32(proj), "chunk_decode: bf16");
  OneRow one;
  const CacheDims c = one_row_dims(k_cache, v_cache, proj, vdim, one);
  const int64_t T = proj.size(0);
  if (q.has_value()) TORCH_CHECK(q->dim() == 3 && q->is_contiguous() && q->is_cuda() && q->scalar_type() == proj.scalar_type() && q->size(0) == T && q->size(1) == nh && q->size(2) == c.dkp + one.rt, "q must be contiguous [T, heads, padded dim]");
  rows2d(proj, proj.scalar_type(), T, std::max({q_off + nh * dim, k_off + c.nkv * dim, v_off + c.nkv * vdim, gate_off + gate_columns(gates, nh, vdim)}), "projections");
  const Extra ex = extra(sink, rel, nh);
  rows2d(out, proj.scalar_type(), T, o_off + nh * vdim, "output");
  TORCH_CHECK(rot_dims == 0 || (cos_t.dim() == 2 && cos_t.size(1) * 2 == rot_dims && cos_t.sizes() == sin_t.sizes()), "rotation tables must be [positions, rot_dims / 2]");
  TORCH_CHECK(block_tables.dim() == 2 && rows.numel() >= 1 && rows.numel() <= T && shares >= 1 && shares <= 64, "block tables [sequences, blocks]; at most T rows; 1 to 64 shares");
  Tensor part;
  if (shares > 1) part = at::empty({rows.numel() * nh * shares * (2 + c.dvp)}, proj.options().dtype(at::kFloat));
  check(kvc_decode(q.has_value() ? q->data_ptr() : nullptr, proj.data_ptr(), proj.stride(0), (int)q_off, (int)k_off, (int)v_off, f32p(bias, nh * dim + c.nkv * (dim + vdim), "bias"),
                   f32p(q_norm, dim, "query norm"), f32p(k_norm, dim, "key norm"), f32p(cos_t, 0, "cos"), f32p(sin_t, 0, "sin"), (int)rot_dims, (float)eps, k_cache.data_ptr(), v_cache.data_ptr(),
                   i32p(block_tables, 1, "block tables"), (int)block_tables.size(1), i32p(rows, 1, "rows"), (int)rows.numel(), i32p(tok_seq, T, "tok_seq"), i32p(positions, T, "positions"),
                   i32p(slots, T, "slots"), proj.data_ptr(), proj.stride(0), (int)gate_off, out.data_ptr(), out.stride(0), (int)o_off, (int)nh, (int)c.nkv, (int)dim, (int)c.dkp, (int)vdim,
                   (int)c.dvp, (int)c.bs, (int)chunk, (int)window, (int)keep, (int)gates, ex.sink, ex.rel, ex.rel_n, (float)scale, (float)out_scale, (int)waves, (int)shares, shares > 1 ? (float*)part.data_ptr() : nullptr, one.scale, (int)one.rt, stream()), "chunk_decode");
}

// ---- latent attention.  cache: [blocks, 1, block size, padded rank]; proj: the layer's projections [T, ...]
struct LatentCache { int64_t blocks, bs, rk; };
LatentCache latent_cache(const Tensor& c, at::ScalarType ty) {
  TORCH_CHECK(c.is_cuda() && c.scalar_type() == ty && c.dim() == 4 && c.size(1) == 1 && c.is_contiguous(), "latent cache: contiguous [blocks, 1, block size, rank] of the activations' type");
  return {c.size(0), c.size(2), c.size(3)};
}

struct Turn { const float* c = nullptr; const float* s = nullptr; int64_t rot = 0; };
Turn turn_tables(const OptT& cos_t, const OptT& sin_t) {
  if (!cos_t.has_value()) return {};
  TORCH_CHECK(sin_t.has_value() && cos_t->dim() == 2 && cos_t->sizes() == sin_t->sizes(), "rotation tables must be [positions, dims / 2]");
  return {f32p(cos_t, 1, "cos"), f32p(sin_t, 1, "sin"), 2 * cos_t->size(1)};
}

// Normed latents into the cache (gain None: it stays).  With cos and sin, the key part (column kr_off) goes behind the latent, rkp elements
// in, and the queries' parts (column r_off + head * padded part) to columns d_off + head d_head of dst.
void latent_write(Tensor proj, int64_t c_off, OptT gain, Tensor slots, Tensor positions, Tensor cache, int64_t rank, int64_t rkp, double eps, int64_t kr_off, OptT cos_t, OptT sin_t, int64_t heads,
                  int64_t r_off, OptT dst, int64_t d_off, int64_t d_head) {
  const bool f = is_f32(proj);
  const LatentCache c = latent_cache(cache, proj.scalar_type());
  const int64_t T = proj.size(0), rtp = c.rk - rkp;
  const Turn tn = turn_tables(cos_t, sin_t);
  TORCH_CHECK(rkp > 0 && rtp >= tn.rot && (tn.rot > 0 || rtp == 0), "latent_write: a cache row is the padded latent and the padded rotated part");
  rows2d(proj, proj.scalar_type(), T, gain.has_value() ? c_off + rkp : 1, "projections");
  if (tn.rot) {
    rows2d(proj, proj.scalar_type(), T, std::max(gain.has_value() ? kr_off + tn.rot : 0, r_off + heads * rtp), "projections");
    TORCH_CHECK(dst.has_value() && d_head >= rtp, "latent_write: rotated queries need a place");
    rows2d(*dst, proj.scalar_type(), T, d_off + (heads - 1) * d_head + rtp, "rotated queries");
  }
  check(kvm_latent_write(proj.data_ptr(), f, proj.stride(0), (int)c_off, f32p(gain, rkp, "latent norm"), i32p(slots, T, "slots"), i32p(positions, T, "positions"), cache.data_ptr(), gain.has_value(),
                         (int)T, (int)rank, (int)rkp, (int)tn.rot, (int)rtp, (int)kr_off, tn.c, tn.s, (int)heads, (int)r_off, dst.has_value() ? dst->data_ptr() : nullptr,
                         dst.has_value() ? dst->stride(0) : 0, (int)d_off, (int)d_head, (float)eps, stream()), "latent_write");
}

// x [T, >= x_off + heads * x_head], w [heads, N, K] row-major, out[t][o_off + h o_head + n], n < n_true; gates per head, or (gate_each) per element
void head_rows(Tensor x, int64_t x_off, int64_t x_head, Tensor w, int64_t n_true, OptT gate, int64_t gate_off, bool gate_each, Tensor out, int64_t o_off, int64_t o_head, double out_scale, Tensor slots) {
  const bool f = is_f32(x);
  TORCH_CHECK(w.dim() == 3 && w.is_contiguous() && w.is_cuda() && w.scalar_type() == x.scalar_type() && x_head >= w.size(2) && n_true <= o_head, "head_rows: weights [heads, N, K]");
  const int64_t T = x.size(0), nh = w.size(0);
  rows2d(x, x.scalar_type(), T, x_off + nh * x_head, "rows");
  rows2d(out, x.scalar_type(), T, o_off + nh * o_head, "output");
  const GateSrc gs = gate_src(gate, gate_off, x, gate_each ? nh * n_true : nh);
  check(kvm_head_rows(x.data_ptr(), f, x.stride(0), (int)x_off, (int)x_head, w.data_ptr(), (int)nh, (int)w.size(1), (int)w.size(2), (int)n_true, gs.p, gs.ld, (int)gate_off, gate_each, out.data_ptr(),
                      out.stride(0), (int)o_off, (int)o_head, (float)out_scale, i32p(slots, T, "slots"), (int)T, stream()), "head_rows");
}

// spans: int32 [3, sequences]: first workspace row, first position, rows
void latent_gather(Tensor cache, Tensor spans, Tensor block_tables, Tensor ws) {
  TORCH_CHECK(!is_f32(ws), "latent_gather: bf16");
  const LatentCache c = latent_cache(cache, ws.scalar_type());
  TORCH_CHECK(ws.dim() == 2 && ws.is_contiguous() && ws.size(1) == c.rk && spans.dim() == 2 && spans.size(0) == 3 && block_tables.dim() == 2 && block_tables.size(0) >= spans.size(1),
              "latent_gather: workspace [rows, rank], spans [3, sequences], block tables [sequences, blocks]");
  const int64_t S = spans.size(1);
  const int* sp = i32p(spans, 3 * S, "spans");
  check(kvl_gather(cache.data_ptr(), ws.data_ptr(), sp, sp + S, sp + 2 * S, (int)S, i32p(block_tables, 1, "block tables"), (int)block_tables.size(1), (int)c.bs, (int)ws.size(0), (int)c.rk, stream()),
        "latent_gather");
}

// kv [workspace rows, heads dkp + heads dvp]; kr [workspace rows, rt]: the keys' rotated parts; blocks: int32 [4, m]: first row, queries
// (0 = unused, at most 128), first position, workspace row of position 0.  Gates per head, or (gate_each) per element.
void latent_prefill(Tensor proj, int64_t q_off, int64_t r_off, int64_t gate_off, bool gate_each, Tensor kv, OptT kr, Tensor blocks, int64_t n_blocks, Tensor out, int64_t o_off, int64_t heads,
                    int64_t dkp, int64_t vdim, int64_t dvp, int64_t window, double scale, double out_scale) {
  TORCH_CHECK(!is_f32(proj), "latent_prefill: bf16");
  const int64_t T = proj.size(0), rt = kr.has_value() ? kr->size(1) : 0;
  rows2d(proj, proj.scalar_type(), T, std::max({q_off + heads * dkp, r_off + heads * rt, gate_off + (gate_each ? heads * vdim : heads)}), "projections");
  rows2d(kv, proj.scalar_type(), 1, heads * (dkp + dvp), "expanded keys and values");
  if (rt) rows2d(*kr, proj.scalar_type(), kv.size(0), rt, "rotated key parts");
  rows2d(out, proj.scalar_type(), T, o_off + heads * vdim, "output");
  TORCH_CHECK(blocks.dim() == 2 && blocks.size(0) == 4, "query blocks [4, n]");
  check(kvl_prefill(proj.data_ptr(), proj.stride(0), (int)q_off, (int)r_off, (int)gate_off, gate_each, kv.data_ptr(), kv.stride(0), (int)(heads * dkp), rt ? kr->data_ptr() : nullptr,
                    rt ? kr->stride(0) : 0, (int)rt, i32p(blocks, 4, "query blocks"), (int)blocks.size(1), (int)n_blocks, out.data_ptr(), out.stride(0), (int)o_off, (int)heads, (int)dkp, (int)vdim,
                    (int)dvp, (int)window, (float)scale, (float)out_scale, stream()), "latent_prefill");
}

// Single tokens (rows, -1 = unused): queries into the latent space, attention there, values and gates.  absorb [heads, rk, dkp] and up
// [heads, dvp, rk] in fragment order; a cache row is rk elements and the rotated part.  write: the rows' latents are normed and written into
// the cache first; turn: the queries' rotated parts are rotated here.
void latent_rows(Tensor proj, int64_t q_off, int64_t r_off, int64_t c_off, int64_t kr_off, int64_t gate_off, bool gate_each, Tensor absorb, Tensor up, OptT c_norm, int64_t rank, double eps, OptT cos_t,
                 OptT sin_t, Tensor cache, bool write, bool turn, Tensor block_tables, Tensor rows, Tensor tok_seq, Tensor positions, Tensor slots, Tensor out, int64_t o_off, int64_t vdim,
                 int64_t window, double scale, double out_scale, int64_t shares, int64_t parts) {
  TORCH_CHECK(!is_f32(proj), "latent_rows: bf16");
  const LatentCache c = latent_cache(cache, proj.scalar_type());
  TORCH_CHECK(absorb.dim() == 3 && up.dim() == 3 && absorb.is_contiguous() && up.is_contiguous() && absorb.scalar_type() == proj.scalar_type() && up.scalar_type() == proj.scalar_type() &&
              absorb.is_cuda() && up.is_cuda() && absorb.size(0) == up.size(0) && absorb.size(1) <= c.rk && up.size(2) == absorb.size(1), "latent_rows: absorb [heads, rank, dim], up [heads, vdim, rank]");
  const int64_t T = proj.size(0), nh = absorb.size(0), rk = absorb.size(1), rt = c.rk - rk, dkp = absorb.size(2), dvp = up.size(1), n = rows.numel();
  const Turn tn = turn_tables(cos_t, sin_t);
  TORCH_CHECK(tn.rot <= rt && (tn.rot > 0) == (rt > 0), "latent_rows: rotation tables and cache rows do not fit");
  rows2d(proj, proj.scalar_type(), T, std::max({q_off + nh * dkp, r_off + nh * rt, write ? std::max(c_off + rk, kr_off + tn.rot) : 0, gate_off + (gate_each ? nh * vdim : nh)}), "projections");
  rows2d(out, proj.scalar_type(), T, o_off + nh * vdim, "output");
  TORCH_CHECK(block_tables.dim() == 2 && n >= 1 && n <= T && shares >= 1 && shares <= 64 && parts >= 1 && parts <= 16, "block tables [sequences, blocks]; at most T rows; 1 to 64 shares");
  const int* rp = i32p(rows, n, "rows");
  const int* sl = i32p(slots, T, "slots");
  const int* ps = i32p(positions, T, "positions");
  Tensor q_lat = at::empty({n, nh, c.rk}, proj.options());
  Tensor lat = at::empty({n, nh, rk}, proj.options()), part;
  if (shares > 1) part = at::empty({n, nh, shares, rk + 4}, proj.options().dtype(at::kFloat));
  check(kvl_absorb(proj.data_ptr(), proj.stride(0), (int)q_off, (int)c_off, absorb.data_ptr(), q_lat.data_ptr(), cache.data_ptr(), write, rp, (int)n, sl, write ? f32p(c_norm, rk, "latent norm") : nullptr,
                   (int)rank, (float)eps, (int)nh, (int)dkp, (int)rk, (int)rt, ps, (int)r_off, (int)kr_off, (int)tn.rot, turn, tn.c, tn.s, stream()), "latent absorb");
  check(kvl_decode(q_lat.data_ptr(), cache.data_ptr(), lat.data_ptr(), shares > 1 ? (float*)part.data_ptr() : nullptr, i32p(block_tables, 1, "block tables"), (int)block_tables.size(1), rp, (int)n,
                   i32p(tok_seq, T, "tok_seq"), ps, sl, (int)nh, (int)rk, (int)rt, (int)c.bs, (int)window, (float)scale, (int)shares, stream()), "latent decode");
  check(kvl_up(lat.data_ptr(), up.data_ptr(), proj.data_ptr(), proj.stride(0), (int)gate_off, gate_each, out.data_ptr(), out.stride(0), (int)o_off, rp, (int)n, sl, (int)nh, (int)rk, (int)vdim,
               (int)dvp, (float)out_scale, (int)parts, stream()), "latent up");
}

// ---- mixture of experts
// router: fp32 [E, K], or bf16 [Ep, K] in fragment order, with one more row for a shared expert's gate; returns (experts int32 [T, top], -1
// in padding rows; weights fp32 [T, top]; the shared expert's gate fp32 [T], or [0]).  scores: 0 sigmoid, 1 softmax, 2 softmax over the chosen;
// bias [E] is added to the logits
std::vector<Tensor> route(Tensor h, Tensor router, Tensor correction, Tensor slots, int64_t top, int64_t scores, double scale, bool shared, OptT bias) {
  const bool f = is_f32(h);
  TORCH_CHECK(router.dim() == 2 && router.is_contiguous() && router.is_cuda() && router.scalar_type() == h.scalar_type(), "route: router [experts, width]");
  const int64_t T = h.size(0), E = correction.numel(), K = router.size(1);
  rows2d(h, h.scalar_type(), T, K, "route: rows");
  TORCH_CHECK(router.size(0) >= E + shared && (!f || router.size(0) == E + shared), "route: router rows");
  Tensor idx = at::empty({T, top}, h.options().dtype(at::kInt)), wt = at::empty({T, top}, h.options().dtype(at::kFloat)), sg = at::empty({shared ? T : 0}, wt.options());
  check(kve_route(h.data_ptr(), f, h.stride(0), router.data_ptr(), f32p(correction, E, "correction"), i32p(slots, T, "slots"), (int)T, (int)E, (int)router.size(0), (int)top, (int)K, (int*)idx.data_ptr(),
                  (float*)wt.data_ptr(), (int)scores, (float)scale, shared ? (float*)sg.data_ptr() : nullptr, f32p(bias, E, "router bias"), stream()), "route");
  return {idx, wt, sg};
}

// The chosen experts' outputs, one row per pair: [T * top, K of gate_up].  gate_up [E, 2 ffp, K] (gated) or [E, ffp, K] (squared relu), down [E, K, ffp].  tile: rows per tile of the
// grouped products (64, 128 or 256), 0: the few-row kernels (bf16: at most 128 tokens).
Tensor expert_outputs(Tensor h, Tensor idx, Tensor gate_up, Tensor down, bool gated, double limit, double slope, double shift, int64_t tile) {
  const bool f = is_f32(h);
  const int64_t T = h.size(0), top = idx.size(1), P = T * top, E = gate_up.size(0), N = gate_up.size(1), K = gate_up.size(2), ffp = gated ? N / 2 : N;
  const int mode = gated ? 1 : 2;
  TORCH_CHECK(gate_up.dim() == 3 && down.dim() == 3 && gate_up.is_contiguous() && down.is_contiguous() && gate_up.is_cuda() && down.is_cuda() && gate_up.scalar_type() == h.scalar_type() &&
              down.scalar_type() == h.scalar_type() && down.size(0) == E && down.size(1) == K && down.size(2) == ffp && (!gated || N % 2 == 0), "experts: gate_up [E, 2 ff, K], down [E, K, ff]");
  TORCH_CHECK(idx.dim() == 2 && idx.size(0) == T, "experts: choices [T, top]");
  rows2d(h, h.scalar_type(), T, K, "experts: rows");
  const int* ip = i32p(idx, P, "choices");
  Tensor act = at::empty({P, ffp}, h.options()), y = at::empty({P, K}, h.options());
  if (tile == 0) {
    check(kve_rows(gate_up.data_ptr(), h.data_ptr(), act.data_ptr(), f, mode, ip, (int)P, (int)top, (int)E, (int)N, (int)K, h.stride(0), ffp, (float)limit, (float)slope, (float)shift, stream()), "expert gate / up");
    check(kve_rows(down.data_ptr(), act.data_ptr(), y.data_ptr(), f, 0, ip, (int)P, (int)top, (int)E, (int)K, (int)ffp, ffp, K, (float)limit, (float)slope, (float)shift, stream()), "expert down");
    return y;
  }
  TORCH_CHECK(!f && (tile == 64 || tile == 128 || tile == 256), "experts: tiles of 64, 128 or 256 rows, bf16");
  const int64_t max_tiles = P / tile + std::min(E, P);
  Tensor ws = at::empty({P + 3 * max_tiles + 1}, idx.options());
  int* order = (int*)ws.data_ptr();
  int* tiles = order + P;
  int* n_tiles = tiles + 3 * max_tiles;
  check(kve_group(ip, (int)P, (int)E, (int)tile, order, tiles, (int)max_tiles, n_tiles, stream()), "expert grouping");
  check(kv_wide_gemm_grouped(gate_up.data_ptr(), h.data_ptr(), act.data_ptr(), (int)N, (int)K, h.stride(0), ffp, mode, (float)limit, (float)slope, (float)shift, (int)tile, order, tiles, (int)max_tiles, n_tiles, (int)top, stream()),
        "grouped gate / up");
  check(kv_wide_gemm_grouped(down.data_ptr(), act.data_ptr(), y.data_ptr(), (int)K, (int)ffp, ffp, K, 0, (float)limit, (float)slope, (float)shift, (int)tile, order, tiles, (int)max_tiles, n_tiles, 1, stream()), "grouped down");
  return y;
}

void argmax_f32(Tensor logits, Tensor out) {
  TORCH_CHECK(logits.is_cuda() && logits.scalar_type() == at::kFloat && logits.dim() == 2 && logits.stride(1) == 1 && out.scalar_type() == at::kLong && out.is_contiguous() &&
              out.numel() >= logits.size(0), "argmax_f32: fp32 [S, V] and int64 [S]");
  check(kvm_argmax_f32((const float*)logits.data_ptr(), logits.stride(0), (int)logits.size(0), (int)logits.size(1), (long long*)out.data_ptr(), stream()), "argmax_f32");
}

// One delta-rule mixer of one layer: its constants, weights and per-sequence state, held for as long as the object lives.
struct DeltaLayer {
  KvdArgs k{};
  Tensor conv_w, a_log, dt_bias, o_norm, state, ring;
  int64_t slots;

  DeltaLayer(int64_t heads, int64_t kv_heads, int64_t dim, int64_t vdim, double eps, double out_scale, std::vector<int64_t> offs, Tensor conv_w_, Tensor a_log_, Tensor dt_bias_, Tensor o_norm_,
             Tensor state_, Tensor ring_)
      : conv_w(conv_w_), a_log(a_log_), dt_bias(dt_bias_), o_norm(o_norm_), state(state_), ring(ring_) {
    TORCH_CHECK(offs.size() == 7, "offsets: q, k, v, beta, decay input, output gate, output");
    TORCH_CHECK(conv_w.dim() == 2 && ring.dim() == 3 && state.dim() == 4 && state.is_contiguous() && ring.is_contiguous() && state.is_cuda() && state.scalar_type() == at::kFloat, "state [slots, heads, dim, vdim] fp32, ring [slots, taps, channels]");
    const int64_t taps = conv_w.size(0), ch = 2 * kv_heads * dim + heads * vdim;
    slots = state.size(0);
    TORCH_CHECK(heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && conv_w.size(1) == ch && ring.size(0) == slots && ring.size(1) == taps && ring.size(2) == ch && state.size(1) == heads &&
                state.size(2) == dim && state.size(3) == vdim, "delta layer: shapes do not fit each other");
    k.q_off = (int)offs[0]; k.k_off = (int)offs[1]; k.v_off = (int)offs[2]; k.b_off = (int)offs[3]; k.z_off = (int)offs[4]; k.gate_off = (int)offs[5]; k.o_off = (int)offs[6];
    k.conv_w = f32p(conv_w, taps * ch, "convolution"); k.a_log = f32p(a_log, heads, "A_log"); k.dt_bias = f32p(dt_bias, heads * dim, "dt_bias"); k.o_norm = f32p(o_norm, vdim, "output norm");
    k.state = (float*)state.data_ptr();
    k.heads = (int)heads; k.kv_heads = (int)kv_heads; k.dim = (int)dim; k.vdim = (int)vdim; k.taps = (int)taps; k.channels = (int)ch;
    k.eps = (float)eps; k.out_scale = (float)out_scale;
  }

  KvdArgs args(const Tensor& proj, const Tensor& low, const OptT& out, const Tensor& tok_seq, const Tensor& positions, const Tensor& tok_kind, const Tensor& tok_off) const {
    KvdArgs a = k;
    const int64_t T = proj.size(0), qk = (int64_t)k.kv_heads * k.dim, v = (int64_t)k.heads * k.vdim;
    TORCH_CHECK(ring.scalar_type() == proj.scalar_type(), "delta layer: the convolution ring has the activations' type");
    rows2d(proj, proj.scalar_type(), T, std::max({k.q_off + qk, k.k_off + qk, k.v_off + v, (int64_t)k.b_off + k.heads}), "projections");
    rows2d(low, proj.scalar_type(), T, std::max((int64_t)k.z_off + (int64_t)k.heads * k.dim, (int64_t)k.gate_off + v), "low-rank projections");
    a.ldp = proj.stride(0); a.ldl = low.stride(0);
    if (out.has_value()) { rows2d(*out, proj.scalar_type(), T, k.o_off + v, "output"); a.ldo = out->stride(0); }
    a.tok_seq = i32p(tok_seq, T, "tok_seq"); a.positions = i32p(positions, T, "positions"); a.tok_kind = i32p(tok_kind, T, "tok_kind"); a.tok_off = i32p(tok_off, T, "tok_off");
    return a;
  }

  bool has_step() const { return kvd_step_rows(k.dim, k.vdim) > 0; }

  bool has_tiles() const { return kvd_tile_dkp(k.dim) > 0; }

  // rows that are the only token of their sequence (-1 = unused): everything in one launch
  void step(Tensor proj, Tensor low, Tensor out, Tensor tok_seq, Tensor positions, Tensor tok_kind, Tensor tok_off, Tensor rows) {
    const KvdArgs a = args(proj, low, out, tok_seq, positions, tok_kind, tok_off);
    TORCH_CHECK(rows.numel() >= 1 && rows.numel() <= proj.size(0), "delta step: at most one listed row per row");
    check(kvd_step(&a, proj.data_ptr(), low.data_ptr(), ring.data_ptr(), out.data_ptr(), is_f32(proj), i32p(rows, 1, "rows"), (int)rows.numel(), stream()), "delta step");
  }

  // segs: int32 [5, n]: first row, tokens, first position, slot, first tile of the portions; those of at least min_n tokens (1 or 2)
  // are served.  tiles: int32 [4, m]: first row, tokens (0 = unused), first position, slot of every 16 tokens of them, the first
  // n_tiles in use at most (0: token by token).
  void portions(Tensor proj, Tensor low, Tensor out, Tensor tok_seq, Tensor positions, Tensor tok_kind, Tensor tok_off, Tensor segs, int64_t min_n, Tensor tiles, int64_t n_tiles) {
    const KvdArgs a = args(proj, low, out, tok_seq, positions, tok_kind, tok_off);
    TORCH_CHECK(segs.dim() == 2 && segs.size(0) == 5 && (min_n == 1 || min_n == 2), "portions: segs [5, n], min_n 1 or 2");
    const int64_t T = proj.size(0), dimp = (k.dim + 7) / 8 * 8, n_segs = segs.size(1);
    const bool f = is_f32(proj);
    auto fo = proj.options().dtype(at::kFloat);
    if (n_tiles > 0) {
      TORCH_CHECK(tiles.dim() == 2 && tiles.size(0) == 4 && n_tiles <= tiles.size(1) && has_tiles(), "portions: tiles [4, m]");
      const int64_t dvp = (k.vdim + 15) / 16 * 16;
      Tensor ws = at::empty({n_tiles * k.heads * (int64_t)kvd_tile_floats(kvd_tile_dkp(k.dim), (int)dvp)}, fo), oc = at::empty({T, k.heads, k.vdim}, fo);
      check(kvd_tiles(&a, proj.data_ptr(), low.data_ptr(), ring.data_ptr(), f, i32p(tiles, 4 * n_tiles, "tiles"), (int)tiles.size(1), (int)n_tiles, i32p(segs, 5 * n_segs, "segs"), (int)n_segs,
                      (int)min_n, (float*)ws.data_ptr(), (float*)oc.data_ptr(), stream()), "delta tiles");
      check(kvd_out(&a, (const float*)oc.data_ptr(), low.data_ptr(), out.data_ptr(), f, (int)min_n, (int)T, stream()), "delta out");
      return;
    }
    Tensor qn = at::empty({T, k.kv_heads, dimp}, fo), kn = at::empty({T, k.kv_heads, dimp}, fo), vv = at::empty({T, k.heads, k.vdim}, fo), dec = at::empty({T, k.heads, dimp}, fo);
    Tensor beta = at::empty({T, k.heads}, fo), o = at::empty({T, k.heads, k.vdim}, fo);
    const int* sp = i32p(segs, 5 * n_segs, "segs");
    auto fp = [](Tensor& t) { return (float*)t.data_ptr(); };
    check(kvd_prep(&a, proj.data_ptr(), low.data_ptr(), ring.data_ptr(), f, fp(qn), fp(kn), fp(vv), fp(dec), fp(beta), (int)dimp, (int)min_n, (int)T, stream()), "delta prep");
    check(kvd_scan(fp(qn), fp(kn), fp(vv), fp(dec), fp(beta), fp(o), sp, (int)n_segs, (int)min_n, (int)dimp, k.state, k.heads, k.kv_heads, k.dim, k.vdim, stream()), "delta scan");
    check(kvd_out(&a, fp(o), low.data_ptr(), out.data_ptr(), f, (int)min_n, (int)T, stream()), "delta out");
    check(kvd_conv_tail(&a, proj.data_ptr(), ring.data_ptr(), f, sp, (int)n_segs, (int)min_n, stream()), "delta conv tail");
  }
};

// One retention mixer of one layer: its constants and per-sequence state, held for as long as the object lives.
struct RetentionLayer {
  KvrArgs k{};
  Tensor log2_decay, cos_t, sin_t, state;

  RetentionLayer(int64_t heads, int64_t dim, int64_t vdim, double eps, double out_scale, std::vector<int64_t> offs, Tensor log2_decay_, Tensor cos_, Tensor sin_, int64_t rot_dims, Tensor state_)
      : log2_decay(log2_decay_), cos_t(cos_), sin_t(sin_), state(state_) {
    TORCH_CHECK(offs.size() == 5, "offsets: q, k, v, gate, output");
    const int64_t dimp = (dim + 15) / 16 * 16, dvp = (vdim + 15) / 16 * 16;
    TORCH_CHECK(heads > 0 && dim > 0 && vdim > 0 && state.is_cuda() && state.scalar_type() == at::kFloat && state.is_contiguous() && state.dim() == 4 && state.size(1) == heads && state.size(2) == dimp &&
                state.size(3) == dvp, "state: fp32 [slots, heads, dim, vdim], sizes rounded up to 16");
    TORCH_CHECK(rot_dims >= 0 && rot_dims <= dim && cos_t.dim() == 2 && cos_t.size(1) * 2 == rot_dims && cos_t.sizes() == sin_t.sizes(), "rotation tables must be [positions, rot_dims / 2]");
    k.q_off = (int)offs[0]; k.k_off = (int)offs[1]; k.v_off = (int)offs[2]; k.g_off = (int)offs[3]; k.o_off = (int)offs[4];
    k.log2_decay = f32p(log2_decay, heads, "decay"); k.cos_t = f32p(cos_t, 0, "cos"); k.sin_t = f32p(sin_t, 0, "sin");
    k.rot_dims = (int)rot_dims; k.heads = (int)heads; k.dim = (int)dim; k.vdim = (int)vdim; k.dimp = (int)dimp; k.dvp = (int)dvp;
    k.k_scale = (float)(1.0 / std::sqrt((double)dim)); k.eps = (float)eps; k.out_scale = (float)out_scale;
    k.state = (float*)state.data_ptr();
  }

  KvrArgs args(const Tensor& proj, const Tensor& out, const Tensor& tok_seq, const Tensor& positions, const Tensor& tok_kind) const {
    KvrArgs a = k;
    const int64_t T = proj.size(0), qk = (int64_t)k.heads * k.dim, v = (int64_t)k.heads * k.vdim;
    rows2d(proj, proj.scalar_type(), T, std::max({k.q_off + qk, k.k_off + qk, k.v_off + v, k.g_off + v}), "projections");
    rows2d(out, proj.scalar_type(), T, k.o_off + v, "output");
    a.ldp = proj.stride(0); a.ldo = out.stride(0);
    a.tok_seq = i32p(tok_seq, T, "tok_seq"); a.positions = i32p(positions, T, "positions"); a.tok_kind = i32p(tok_kind, T, "tok_kind");
    return a;
  }

  bool chunked() const { return kvr_chunked(k.vdim) != 0; }

  // rows that are the only token of their sequence (-1 = unused)
  void step(Tensor proj, Tensor out, Tensor tok_seq, Tensor positions, Tensor tok_kind, Tensor rows) {
    const KvrArgs a = args(proj, out, tok_seq, positions, tok_kind);
    TORCH_CHECK(rows.numel() >= 1 && rows.numel() <= proj.size(0), "retention: at most one listed row per row");
    check(kvr_rows(&a, proj.data_ptr(), out.data_ptr(), is_f32(proj), i32p(rows, 1, "rows"), (int)rows.numel(), stream()), "retention step");
  }

  // segs: int32 [5, n]: first row, tokens, first position, slot of the portions; those of at least two tokens are served.  chunks: int32 [4, m]:
  // first row, tokens (0 = unused), first position of their pieces of 64, the first n_chunks in use at most (0: token by token);
  // first_chunk [n].
  void portions(Tensor proj, Tensor out, Tensor tok_seq, Tensor positions, Tensor tok_kind, Tensor segs, Tensor chunks, int64_t n_chunks, Tensor first_chunk) {
    const KvrArgs a = args(proj, out, tok_seq, positions, tok_kind);
    TORCH_CHECK(segs.dim() == 2 && segs.size(0) == 5 && chunks.dim() == 2 && chunks.size(0) == 4 && n_chunks >= 0 && n_chunks <= chunks.size(1), "portions: segs [5, n], chunks [4, m]");
    const int64_t n = segs.size(1);
    Tensor ws;
    if (n_chunks > 0) ws = at::empty({n_chunks, k.heads, k.dimp, k.dvp}, proj.options().dtype(at::kFloat));
    check(kvr_portions(&a, proj.data_ptr(), out.data_ptr(), is_f32(proj), i32p(segs, 5 * n, "segs"), (int)n, i32p(chunks, 4, "chunks"), (int)chunks.size(1), (int)n_chunks,
                       i32p(first_chunk, n, "first chunks"), n_chunks > 0 ? (float*)ws.data_ptr() : nullptr, stream()), "retention portions");
  }
};

// One state-space mixer of one layer: its constants, weights and per-sequence memory, held for as long as the object lives.
struct StateSpaceLayer {
  KvsArgs k{};
  Tensor conv_w, conv_b, dt_bias, a_log, skip, norm, state, ring;

  StateSpaceLayer(int64_t heads, int64_t groups, int64_t dim, int64_t vdim, int64_t norm_groups, double eps, double out_scale, std::vector<int64_t> offs, Tensor conv_w_, Tensor conv_b_, Tensor dt_bias_,
                  Tensor a_log_, Tensor skip_, Tensor norm_, Tensor state_, Tensor ring_)
      : conv_w(conv_w_), conv_b(conv_b_), dt_bias(dt_bias_), a_log(a_log_), skip(skip_), norm(norm_), state(state_), ring(ring_) {
    TORCH_CHECK(offs.size() == 4, "offsets: gates, channels, steps, output");
    TORCH_CHECK(heads > 0 && groups > 0 && heads % groups == 0 && dim > 0 && vdim > 0 && norm_groups > 0 && heads * vdim % norm_groups == 0, "state space: bad sizes");
    const int64_t dimp = (dim + 15) / 16 * 16, dvp = (vdim + 15) / 16 * 16, ch = heads * vdim + 2 * groups * dim;
    TORCH_CHECK(conv_w.dim() == 2 && conv_w.size(1) == ch && state.is_cuda() && state.scalar_type() == at::kFloat && state.is_contiguous() && state.dim() == 4 && state.size(1) == heads && state.size(2) == dimp &&
                state.size(3) == dvp && ring.is_cuda() && ring.is_contiguous() && ring.dim() == 3 && ring.size(0) == state.size(0) && ring.size(1) == conv_w.size(0) && ring.size(2) == ch,
                "state: fp32 [slots, heads, dim, vdim], sizes rounded up to 16; ring [slots, taps, channels]");
    k.z_off = (int)offs[0]; k.x_off = (int)offs[1]; k.dt_off = (int)offs[2]; k.o_off = (int)offs[3];
    k.taps = (int)conv_w.size(0); k.channels = (int)ch;
    k.conv_w = f32p(conv_w, k.taps * ch, "convolution"); k.conv_b = f32p(conv_b, ch, "convolution bias"); k.dt_bias = f32p(dt_bias, heads, "dt_bias"); k.a_log = f32p(a_log, heads, "A_log");
    k.skip = f32p(skip, heads, "D"); k.norm = f32p(norm, heads * vdim, "norm");
    k.heads = (int)heads; k.groups = (int)groups; k.dim = (int)dim; k.vdim = (int)vdim; k.dimp = (int)dimp; k.dvp = (int)dvp; k.norm_groups = (int)norm_groups;
    k.eps = (float)eps; k.out_scale = (float)out_scale;
    k.state = (float*)state.data_ptr();
  }

  // rows: the ones that are the only token of their sequence (-1 = unused).  With n_chunks > 0 also the portions of several tokens: segs int32
  // [5, n]: first row, tokens, first position, slot; chunks int32 [4, m]: first row, tokens (0 = unused) of their pieces of 64, the first
  // n_chunks in use at most; first_chunk [n].
  void run(Tensor proj, Tensor out, Tensor tok_seq, Tensor positions, Tensor tok_kind, Tensor tok_off, Tensor rows, Tensor segs, OptT chunks, int64_t n_chunks, OptT first_chunk) {
    KvsArgs a = k;
    const bool f = is_f32(proj);
    const int64_t T = proj.size(0), inner = (int64_t)k.heads * k.vdim;
    rows2d(proj, proj.scalar_type(), T, std::max({k.z_off + inner, (int64_t)k.x_off + k.channels, (int64_t)k.dt_off + k.heads}), "projections");
    rows2d(out, proj.scalar_type(), T, k.o_off + inner, "output");
    TORCH_CHECK(ring.scalar_type() == proj.scalar_type(), "state space: the convolution's last inputs have the activations' type");
    TORCH_CHECK(rows.numel() >= 1 && rows.numel() <= T, "state space: at most one listed row per row");
    a.ldp = proj.stride(0); a.ldo = out.stride(0);
    a.tok_seq = i32p(tok_seq, T, "tok_seq"); a.positions = i32p(positions, T, "positions"); a.tok_kind = i32p(tok_kind, T, "tok_kind"); a.tok_off = i32p(tok_off, T, "tok_off");
    auto fo = proj.options().dtype(at::kFloat);
    Tensor y = at::empty({T, inner}, fo);
    check(kvs_step(&a, proj.data_ptr(), ring.data_ptr(), (float*)y.data_ptr(), f, i32p(rows, 1, "rows"), (int)rows.numel(), stream()), "state-space step");
    if (n_chunks > 0) {
      TORCH_CHECK(chunks.has_value() && first_chunk.has_value() && segs.dim() == 2 && segs.size(0) == 5 && chunks->dim() == 2 && chunks->size(0) == 4 && n_chunks <= chunks->size(1),
                  "state space: segs [5, n], chunks [4, m]");
      const int64_t n = segs.size(1);
      Tensor xbc = at::empty({T, k.channels}, proj.options()), ws = at::empty({(int64_t)kvs_workspace(&a, (int)T, (int)n_chunks)}, fo);
      check(kvs_portions(&a, proj.data_ptr(), ring.data_ptr(), (float*)y.data_ptr(), f, xbc.data_ptr(), (float*)ws.data_ptr(), (int)T, i32p(segs, 5 * n, "segs"), (int)n, i32p(*chunks, 4, "chunks"),
                         (int)chunks->size(1), (int)n_chunks, i32p(*first_chunk, n, "first chunks"), stream()), "state-space portions");
    }
    check(kvs_gate(&a, proj.data_ptr(), (const float*)y.data_ptr(), out.data_ptr(), f, (int)T, stream()), "state-space gate");
  }
};

}  // namespace

void bind_mixers(pybind11::module_& m) {
  namespace py = pybind11;
  m.def("embed_stream", &embed_stream);
  m.def("gated_residual", &gated_residual);
  m.def("hyper_residual", &hyper_residual);
  m.def("parallel_residual", &parallel_residual);
  m.def("softcap", &softcap);
  m.def("norm_rope_write", &norm_rope_write);
  m.def("row_attention", &row_attention);
  m.def("chunk_prefill", &chunk_prefill);
  m.def("chunk_prefill_supported", [](int64_t dkp, int64_t dvp) { return kvc_supported((int)dkp, (int)dvp) != 0; });
  m.def("chunk_decode", &chunk_decode);
  m.def("key_value_write", &key_value_write);
  m.def("argmax_f32", &argmax_f32);
  m.def("latent_supported", [](int64_t dkp, int64_t dvp, int64_t rk) { return kvl_supported((int)dkp, (int)dvp, (int)rk) != 0; });
  m.def("latent_write", &latent_write);
  m.def("head_rows", &head_rows);
  m.def("latent_gather", &latent_gather);
  m.def("latent_prefill", &latent_prefill);
  m.def("latent_rows", &latent_rows);
  m.def("route", &route);
  m.def("expert_outputs", &expert_outputs);
  py::class_<DeltaLayer>(m, "DeltaLayer")
      .def(py::init<int64_t, int64_t, int64_t, int64_t, double, double, std::vector<int64_t>, Tensor, Tensor, Tensor, Tensor, Tensor, Tensor>())
      .def("has_step", &DeltaLayer::has_step)
      .def("has_tiles", &DeltaLayer::has_tiles)
      .def("step", &DeltaLayer::step)
      .def("portions", &DeltaLayer::portions);
  py::class_<RetentionLayer>(m, "RetentionLayer")
      .def(py::init<int64_t, int64_t, int64_t, double, double, std::vector<int64_t>, Tensor, Tensor, Tensor, int64_t, Tensor>())
      .def("chunked", &RetentionLayer::chunked)
      .def("step", &RetentionLayer::step)
      .def("portions", &RetentionLayer::portions);
  py::class_<StateSpaceLayer>(m, "StateSpaceLayer")
      .def(py::init<int64_t, int64_t, int64_t, int64_t, int64_t, double, double, std::vector<int64_t>, Tensor, Tensor, Tensor, Tensor, Tensor, Tensor, Tensor, Tensor>())
      .def("run", &StateSpaceLayer::run);
}
