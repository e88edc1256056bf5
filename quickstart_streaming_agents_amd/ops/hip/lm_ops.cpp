// Torch bindings of the decoder-mixer kernels (module qsa_lm_hip).  Every
// binding checks shapes, types and strides against what its kernel and grid
// assume; the matrix-core variants are chosen here where the sizes fit them.
#include <hip/hip_runtime.h>
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

typedef unsigned short bf16_t;

#define CHK_DEV(t) TORCH_CHECK((t).is_cuda(), #t " must be on the GPU")
#define CHK_CONT(t) TORCH_CHECK((t).is_contiguous(), #t " must be contiguous")
#define CHK_F32(t) TORCH_CHECK((t).scalar_type() == at::kFloat && (t).is_contiguous(), #t " must be contiguous f32")
#define CHK_I32(t) TORCH_CHECK((t).scalar_type() == at::kInt && (t).is_contiguous(), #t " must be contiguous i32")
#define CHK_SAME(a, b) TORCH_CHECK((a).scalar_type() == (b).scalar_type(), #a " and " #b " must have one dtype")

using torch::Tensor;
using OptTensor = c10::optional<Tensor>;

static inline hipStream_t cur_stream() {
  return at::hip::getCurrentHIPStream().stream();
}
static inline int is_f32(const Tensor& t) {
  TORCH_CHECK(t.scalar_type() == at::kFloat || t.scalar_type() == at::kBFloat16,
              "bf16 or f32 expected");
  return t.scalar_type() == at::kFloat;
}
static inline bool aligned(const Tensor& t, int bytes) {
  return reinterpret_cast<uintptr_t>(t.data_ptr()) % bytes == 0;
}
static inline void chk_rows(const Tensor& t, const char* name) {
  TORCH_CHECK(t.dim() == 2 && t.stride(1) == 1, name,
              " must be 2-D with contiguous rows");
}
static inline const bf16_t* u16(const Tensor& t) {
  return reinterpret_cast<const bf16_t*>(t.data_ptr());
}
static inline bf16_t* u16m(const Tensor& t) {
  return reinterpret_cast<bf16_t*>(t.data_ptr());
}

// a step's rows for the short convolutions (ops/hip/short_conv.hip)
struct ConvStep {
  const int *item, *t0, *off, *start, *len, *slots;
};

extern "C" void qsa_residual_norm_launch(float*, const void*, long long,
    const void*, const void*, const long long*, float, const void*,
    const void*, const void*, void*, long long, int, int, float, int, int,
    int, int, hipStream_t);
extern "C" void qsa_glu_launch(const void*, const void*, const long long*,
    void*, long long, long long, long long, long long, long long, int, int,
    int, hipStream_t);
extern "C" void qsa_conv_qkv_launch(const void*, long long, const float*, int,
    void*, ConvStep, int, const float*, const float*, int, int, const int*,
    void*, void*, void*, int, int, int, int, int, int, hipStream_t);
extern "C" void qsa_conv_silu_launch(const void*, long long, const float*,
    const float*, int, void*, ConvStep, int, void*, int, int, int,
    hipStream_t);
extern "C" void qsa_gqa_rows_launch(const void*, const void*, const void*,
    const int*, int, const int*, const int*, const float*, const void*,
    long long, void*, long long, int, int, int, int, int, float, float, int,
    hipStream_t);
extern "C" void qsa_gqa_rows_mfma_launch(const bf16_t*, const bf16_t*,
    const bf16_t*, const int*, int, const int*, const int*, const float*,
    const bf16_t*, long long, float*, float*, bf16_t*, long long, int, int,
    int, int, int, float, float, int, hipStream_t);
extern "C" void qsa_gqa_portions_launch(const bf16_t*, const bf16_t*,
    const bf16_t*, const int*, int, const float*, const bf16_t*, long long,
    const int*, const int*, const int*, const int*, const int*, bf16_t*,
    long long, int, int, int, int, int, float, float, int, hipStream_t);
extern "C" void qsa_ssd_decode_launch(const void*, long long, int, int,
    const void*, const float*, const float*, const float*, float*, const int*,
    const int*, void*, int, int, int, int, int, int, int, hipStream_t);
extern "C" void qsa_ssd_seq_launch(const void*, long long, int, int,
    const void*, const float*, const float*, const float*, float*, const int*,
    const int*, const int*, const int*, void*, int, int, int, int, int, int,
    hipStream_t);
extern "C" void qsa_ssd_steps_launch(const bf16_t*, long long, int,
    const float*, const float*, const int*, const int*, const int*,
    const int*, float*, int, int, hipStream_t);
extern "C" void qsa_ssd_state_launch(const bf16_t*, const float*, float*,
    const int*, const int*, const int*, const int*, const int*, void*, int,
    int, int, int, int, int, int, hipStream_t);
extern "C" void qsa_ssd_out_launch(const bf16_t*, long long, int,
    const bf16_t*, const float*, const float*, const int*, const int*,
    const int*, const int*, const int*, const void*, int, bf16_t*, int, int,
    int, int, int, int, hipStream_t);
extern "C" void qsa_part_norm_launch(const void*, const float*, void*,
    long long, long long, int, int, float, int, int, hipStream_t);
extern "C" void qsa_latent_norm_store_launch(const void*, long long,
    const void*, const void*, void*, void*, const int*, long long, int, int,
    float, int, hipStream_t);
extern "C" void qsa_decode_slots_launch(const int*, const int*, int*, int,
    int, hipStream_t);
extern "C" void qsa_argmax_rows_launch(const void*, long long*, long long,
    int, int, hipStream_t);
extern "C" void qsa_retention_decode_launch(const void*, long long,
    const float*, const float*, const float*, float*, const int*, const int*,
    void*, int, int, int, int, int, float, float, int, int, int, hipStream_t);
extern "C" void qsa_retention_seq_launch(const void*, long long,
    const float*, const float*, const float*, float*, const int*, const int*,
    const int*, const int*, void*, int, int, int, int, int, float, float,
    int, int, hipStream_t);
extern "C" void qsa_retention_rotate_launch(const bf16_t*, long long,
    const float*, const float*, const int*, bf16_t*, long long, int, int,
    int, int, float, int, hipStream_t);
extern "C" void qsa_retention_state_launch(const bf16_t*, long long,
    long long, const bf16_t*, long long, const float*, float*, const int*,
    const int*, const int*, const int*, const int*, void*, int, int, int,
    int, int, int, hipStream_t);
extern "C" void qsa_retention_out_launch(const bf16_t*, long long, long long,
    const bf16_t*, long long, const float*, const int*, const int*,
    const int*, const int*, const int*, const void*, long long, bf16_t*,
    int, int, int, int, float, hipStream_t);
extern "C" void qsa_head_matmul_launch(const void*, long long, const void*,
    const void*, long long, void*, int, int, int, int, int, int, hipStream_t);
extern "C" void qsa_latent_rows_launch(const void*, const void*, const int*,
    int, const int*, const int*, const void*, void*, int, int, int, int,
    float, int, hipStream_t);
extern "C" void qsa_latent_rows_mfma_launch(const bf16_t*, const bf16_t*,
    const int*, int, const int*, const int*, const bf16_t*, float*, float*,
    bf16_t*, int, int, int, int, float, int, hipStream_t);
extern "C" void qsa_window_attn_prefill_launch(const bf16_t*, long long,
    const bf16_t*, long long, const bf16_t*, long long, const bf16_t*,
    const int*, const int*, const int*, const int*, const int*, const int*,
    const int*, bf16_t*, int, int, int, int, int, float, hipStream_t);
extern "C" void qsa_skinny_gemm_launch(const bf16_t*, const bf16_t*, bf16_t*,
    int, int, long long, long long, hipStream_t);

// res [T, W] f32 updated in place; returns norm(res) * w (+ b), or res itself
// in y's storage type when w is not given
Tensor residual_norm(Tensor res, OptTensor y, OptTensor table, OptTensor ids,
                     OptTensor vec, OptTensor w, OptTensor b, double eps,
                     bool init, bool layer, OptTensor post, double tscale) {
  CHK_DEV(res); CHK_F32(res);
  TORCH_CHECK(res.dim() == 2, "res [T, W]");
  TORCH_CHECK(w || y, "norm weight or y");
  const long long T = res.size(0);
  const int W = (int)res.size(1);
  const Tensor& like = w ? *w : *y;
  const int f32 = is_f32(like);
  auto out = torch::empty({T, (long long)W}, like.options());
  if (T == 0) return out;
  bool v4 = W % 4 == 0;
  const int word = f32 ? 16 : 8;
  auto row_vec = [&](const OptTensor& t, const char* name) -> const void* {
    if (!t) return nullptr;
    CHK_SAME(*t, like); CHK_CONT(*t);
    TORCH_CHECK(t->numel() == W, name, " size");
    v4 = v4 && aligned(*t, word);
    return t->data_ptr();
  };
  const void* wp = row_vec(w, "norm weight");
  const void* bp = row_vec(b, "bias");
  const void* vp = row_vec(vec, "vec");
  const void* pp = row_vec(post, "post-norm weight");
  TORCH_CHECK(!post || y, "post needs y");
  TORCH_CHECK(w || !b, "bias without weight");
  const void *yp = nullptr, *tp = nullptr;
  long long ys = 0;
  int vocab = 0;
  const long long* ip = nullptr;
  if (y) {
    CHK_SAME(*y, like); chk_rows(*y, "y");
    TORCH_CHECK(y->size(0) == T && y->size(1) == W, "y shape");
    yp = y->data_ptr(); ys = y->stride(0);
    v4 = v4 && ys % 4 == 0 && aligned(*y, word);
  }
  if (table) {
    TORCH_CHECK(ids.has_value(), "table needs ids");
    CHK_SAME(*table, like); CHK_CONT(*table); CHK_CONT(*ids);
    TORCH_CHECK(ids->scalar_type() == at::kLong && ids->numel() == T, "ids");
    TORCH_CHECK(table->dim() == 2 && table->size(1) == W, "table shape");
    tp = table->data_ptr(); vocab = (int)table->size(0);
    ip = reinterpret_cast<const long long*>(ids->data_ptr<int64_t>());
    v4 = v4 && aligned(*table, word);
  }
  qsa_residual_norm_launch(res.data_ptr<float>(), yp, ys, pp, tp, ip,
                           (float)tscale, vp, wp, bp, out.data_ptr(), T, W,
                           vocab, (float)eps, init, layer, f32, v4,
                           cur_stream());
  return out;
}

Tensor glu(Tensor gate, Tensor up, bool gelu) {
  CHK_DEV(gate); chk_rows(gate, "gate"); chk_rows(up, "up");
  CHK_SAME(gate, up);
  TORCH_CHECK(gate.sizes() == up.sizes(), "gate/up shapes must match");
  const long long rows = gate.size(0), cols = gate.size(1);
  auto out = torch::empty({rows, cols}, gate.options());
  if (rows == 0 || cols == 0) return out;
  const int v = cols % 8 == 0 && gate.stride(0) % 8 == 0 &&
                up.stride(0) % 8 == 0 && aligned(gate, 16) && aligned(up, 16);
  qsa_glu_launch(gate.data_ptr(), up.data_ptr(), nullptr, out.data_ptr(),
                 rows, cols, gate.stride(0), up.stride(0), 0, gelu,
                 is_f32(gate), v, cur_stream());
  return out;
}

// act(gate [T, n]) * table[ids, col0 : col0 + n]
Tensor glu_table(Tensor gate, Tensor table, Tensor ids, long col0,
                 bool gelu) {
  CHK_DEV(gate); chk_rows(gate, "gate"); CHK_CONT(table); CHK_CONT(ids);
  CHK_SAME(gate, table);
  const long long rows = gate.size(0), cols = gate.size(1);
  TORCH_CHECK(ids.scalar_type() == at::kLong && ids.numel() == rows, "ids");
  TORCH_CHECK(table.dim() == 2 && col0 >= 0 && table.size(0) > 0 &&
                  col0 + cols <= table.size(1), "columns of the table");
  auto out = torch::empty({rows, cols}, gate.options());
  if (rows == 0 || cols == 0) return out;
  const int v = cols % 8 == 0 && gate.stride(0) % 8 == 0 && col0 % 8 == 0 &&
                table.size(1) % 8 == 0 && aligned(gate, 16) &&
                aligned(table, 16);
  const char* base = reinterpret_cast<const char*>(table.data_ptr()) +
                     col0 * table.element_size();
  qsa_glu_launch(gate.data_ptr(), base,
                 reinterpret_cast<const long long*>(ids.data_ptr<int64_t>()),
                 out.data_ptr(), rows, cols, gate.stride(0), table.size(1),
                 table.size(0), gelu, is_f32(gate), v, cur_stream());
  return out;
}

// x [T, >= qr+kr]; returns rms(x[:, :qr]) * wq; the latent goes to the cache
Tensor latent_norm_store(Tensor x, Tensor wq, Tensor wk, Tensor cache,
                         Tensor slots, double eps) {
  CHK_DEV(x); chk_rows(x, "x"); CHK_CONT(wq); CHK_CONT(wk); CHK_CONT(cache);
  CHK_SAME(x, wq); CHK_SAME(x, wk); CHK_SAME(x, cache); CHK_I32(slots);
  const long long T = x.size(0);
  const int qr = (int)wq.numel(), kr = (int)wk.numel();
  TORCH_CHECK(x.size(1) >= qr + kr, "x holds [q latent | kv latent]");
  TORCH_CHECK(cache.dim() == 3 && cache.size(1) == 64 && cache.size(2) == kr,
              "latent cache [pages, 64, kr]");
  TORCH_CHECK(slots.numel() == T, "one slot per row");
  auto cq = torch::empty({T, (long long)qr}, x.options());
  if (T == 0) return cq;
  qsa_latent_norm_store_launch(x.data_ptr(), x.stride(0), wq.data_ptr(),
                               wk.data_ptr(), cq.data_ptr(),
                               cache.data_ptr(), slots.data_ptr<int>(), T, qr,
                               kr, (float)eps, is_f32(x), cur_stream());
  return cq;
}

Tensor decode_slots(Tensor block_table, Tensor seq_lens) {
  CHK_DEV(block_table); CHK_I32(block_table); CHK_I32(seq_lens);
  const int B = (int)seq_lens.numel();
  TORCH_CHECK(block_table.dim() == 2 && block_table.size(0) == B, "table rows");
  auto slots = torch::empty({B}, seq_lens.options());
  if (B)
    qsa_decode_slots_launch(block_table.data_ptr<int>(),
                            seq_lens.data_ptr<int>(), slots.data_ptr<int>(),
                            B, (int)block_table.size(1), cur_stream());
  return slots;
}

Tensor argmax_rows(Tensor x) {
  CHK_DEV(x); CHK_CONT(x);
  TORCH_CHECK(x.dim() == 2 && x.size(1) > 0, "x [rows, n]");
  auto out = torch::empty({x.size(0)}, x.options().dtype(at::kLong));
  if (x.size(0))
    qsa_argmax_rows_launch(x.data_ptr(),
                           reinterpret_cast<long long*>(out.data_ptr<int64_t>()),
                           x.size(0), (int)x.size(1), is_f32(x),
                           cur_stream());
  return out;
}

// ---- retention -------------------------------------------------------------
struct RetDims { int H, D, E, rot, table_len; };

static RetDims ret_check(const Tensor& x, const Tensor& cos_t,
                         const Tensor& sin_t, const Tensor& decay,
                         const Tensor& state, long rot) {
  CHK_DEV(x); chk_rows(x, "x"); CHK_F32(state); CHK_F32(decay);
  TORCH_CHECK(state.dim() == 4, "state [slots, H, D, E]");
  RetDims r{(int)state.size(1), (int)state.size(2), (int)state.size(3),
            (int)rot, 0x7fffffff};
  TORCH_CHECK(decay.numel() == r.H, "one decay per head");
  TORCH_CHECK(x.size(1) >= 2LL * r.H * r.D + 2LL * r.H * r.E,
              "x holds [q | k | v | gate]");
  TORCH_CHECK(rot % 2 == 0 && rot >= 0 && rot <= r.D, "rotated dims");
  if (rot > 0) {
    CHK_F32(cos_t); CHK_F32(sin_t);
    TORCH_CHECK(cos_t.dim() == 2 && cos_t.size(1) == rot / 2 &&
                    sin_t.sizes() == cos_t.sizes(), "rotation tables");
    r.table_len = (int)cos_t.size(0);
  }
  return r;
}

Tensor retention_decode(Tensor x, Tensor cos_t, Tensor sin_t, Tensor decay,
                        Tensor state, Tensor slots, Tensor seq_lens, long rot,
                        double kscale, double eps) {
  const RetDims r = ret_check(x, cos_t, sin_t, decay, state, rot);
  CHK_I32(slots); CHK_I32(seq_lens);
  const int B = (int)x.size(0);
  TORCH_CHECK(slots.numel() == B && seq_lens.numel() == B, "slots/seq_lens");
  TORCH_CHECK(2 * r.D + 2 * r.E <= 8000, "head too wide for the decode block");
  auto out = torch::empty({B, (long long)r.H * r.E}, x.options());
  if (B == 0) return out;
  const int v4 = r.E % 4 == 0 && (2LL * r.H * r.D) % 4 == 0 &&
                 x.stride(0) % 4 == 0 && aligned(x, 16);
  qsa_retention_decode_launch(
      x.data_ptr(), x.stride(0), cos_t.data_ptr<float>(),
      sin_t.data_ptr<float>(), decay.data_ptr<float>(),
      state.data_ptr<float>(), slots.data_ptr<int>(),
      seq_lens.data_ptr<int>(), out.data_ptr(), B, r.H, r.D, r.E, r.rot,
      (float)kscale, (float)eps, r.table_len, is_f32(x), v4, cur_stream());
  return out;
}

static int chk_items(const Tensor& slots, const Tensor& off,
                     const Tensor& start, const Tensor& len) {
  CHK_I32(slots); CHK_I32(off); CHK_I32(start); CHK_I32(len);
  const int n = (int)slots.numel();
  TORCH_CHECK(off.numel() == n && start.numel() == n && len.numel() == n,
              "per-portion arrays");
  return n;
}

// rows of x outside the portions are left unwritten in `out`
void retention_seq(Tensor x, Tensor cos_t, Tensor sin_t, Tensor decay,
                   Tensor state, Tensor slots, Tensor off, Tensor start,
                   Tensor len, Tensor out, long rot, double kscale,
                   double eps) {
  const RetDims r = ret_check(x, cos_t, sin_t, decay, state, rot);
  const int n = chk_items(slots, off, start, len);
  CHK_SAME(x, out); CHK_CONT(out);
  TORCH_CHECK(out.size(0) == x.size(0) && out.size(1) == (long long)r.H * r.E,
              "out [T, H*E]");
  TORCH_CHECK(2 * r.D + r.E <= 12000, "head too wide");
  if (n == 0) return;
  qsa_retention_seq_launch(
      x.data_ptr(), x.stride(0), cos_t.data_ptr<float>(),
      sin_t.data_ptr<float>(), decay.data_ptr<float>(),
      state.data_ptr<float>(), slots.data_ptr<int>(), off.data_ptr<int>(),
      start.data_ptr<int>(), len.data_ptr<int>(), out.data_ptr(), n, r.H, r.D,
      r.E, r.rot, (float)kscale, (float)eps, r.table_len, is_f32(x),
      cur_stream());
}

static int pad_dim(int d) {
  int p = 32;
  while (p < d) p *= 2;
  return p;
}

bool retention_chunked_ok(long H, long D, long E) {
  return D <= 256 && E <= 512 && E % 8 == 0 && (2 * H * D) % 8 == 0 &&
         (H * E) % 8 == 0;
}

// chunked prefill of the portions; rows r0.. of x are the portions' rows
void retention_chunked(Tensor x, Tensor cos_t, Tensor sin_t,
                       Tensor log2_decay, Tensor state, Tensor slots,
                       Tensor off, Tensor start, Tensor len,
                       Tensor positions, Tensor chunk0, Tensor chunk_item,
                       Tensor chunk_t0, Tensor out, long rot, double kscale,
                       double eps) {
  const RetDims r = ret_check(x, cos_t, sin_t, log2_decay, state, rot);
  const int n = chk_items(slots, off, start, len);
  CHK_SAME(x, out); CHK_CONT(out); CHK_I32(positions); CHK_I32(chunk0);
  CHK_I32(chunk_item); CHK_I32(chunk_t0);
  TORCH_CHECK(x.scalar_type() == at::kBFloat16, "bf16 storage");
  TORCH_CHECK(retention_chunked_ok(r.H, r.D, r.E), "sizes of the chunked path");
  TORCH_CHECK(x.stride(0) % 8 == 0 && aligned(x, 16), "x alignment");
  const long long T = x.size(0), nc = chunk_item.numel();
  TORCH_CHECK(positions.numel() == T && chunk0.numel() == n &&
                  chunk_t0.numel() == nc, "plan arrays");
  TORCH_CHECK(out.size(0) == T && out.size(1) == (long long)r.H * r.E, "out");
  if (n == 0 || nc == 0) return;
  const int DP = pad_dim(r.D), EP = (r.E + 15) / 16 * 16;
  auto planes = torch::empty({4, T, r.H, DP}, x.options());
  auto prefix = torch::empty({nc, r.H, 2, EP, DP}, x.options());
  hipStream_t st = cur_stream();
  const long long voff = 2LL * r.H * r.D;
  qsa_retention_rotate_launch(u16(x), x.stride(0), cos_t.data_ptr<float>(),
                              sin_t.data_ptr<float>(),
                              positions.data_ptr<int>(), u16m(planes), T, r.H,
                              r.D, DP, r.rot, (float)kscale, r.table_len, st);
  qsa_retention_state_launch(u16(x), x.stride(0), voff, u16(planes), T,
                             log2_decay.data_ptr<float>(),
                             state.data_ptr<float>(), slots.data_ptr<int>(),
                             off.data_ptr<int>(), start.data_ptr<int>(),
                             len.data_ptr<int>(), chunk0.data_ptr<int>(),
                             prefix.data_ptr(), n, r.H, r.D, DP, r.E, EP, st);
  qsa_retention_out_launch(u16(x), x.stride(0), voff, u16(planes), T,
                           log2_decay.data_ptr<float>(), off.data_ptr<int>(),
                           start.data_ptr<int>(), len.data_ptr<int>(),
                           chunk_item.data_ptr<int>(),
                           chunk_t0.data_ptr<int>(), prefix.data_ptr(), nc,
                           u16m(out), r.H, DP, r.E, EP, (float)eps, st);
}

// ---- latent attention ------------------------------------------------------
// x [M, H, K] rows (row stride free), W [H, N, K] -> [M, H*N]
Tensor head_matmul(Tensor x, Tensor W, OptTensor gate) {
  CHK_DEV(x); chk_rows(x, "x"); CHK_CONT(W); CHK_SAME(x, W);
  TORCH_CHECK(W.dim() == 3, "W [H, N, K]");
  const int H = (int)W.size(0), N = (int)W.size(1), K = (int)W.size(2);
  TORCH_CHECK(x.size(1) == (long long)H * K, "x [M, H*K]");
  TORCH_CHECK(K <= 16000, "K");
  const int M = (int)x.size(0);
  auto out = torch::empty({M, (long long)H * N}, x.options());
  if (M == 0) return out;
  const int f32 = is_f32(x);
  int mfma = !f32 && K % 8 == 0 && N % 4 == 0 && x.stride(0) % 8 == 0 &&
             aligned(x, 16) && aligned(W, 16);
  const void* gp = nullptr;
  long long gs = 0;
  if (gate) {
    CHK_SAME(x, *gate); chk_rows(*gate, "gate");
    TORCH_CHECK(gate->size(0) == M && gate->size(1) == (long long)H * N,
                "gate [M, H*N]");
    gp = gate->data_ptr(); gs = gate->stride(0);
    mfma = mfma && gs % 4 == 0 && aligned(*gate, 8);
  }
  qsa_head_matmul_launch(x.data_ptr(), x.stride(0), W.data_ptr(), gp, gs,
                         out.data_ptr(), M, H, N, K, f32, mfma, cur_stream());
  return out;
}

// qa [R, H*KR] absorbed queries -> normalized latent read-out [R, H*KR].
// row_item: which block_table row a query row uses (none: its own index);
// row_len: position + 1 of the query row (0: row not in use).
Tensor latent_rows(Tensor qa, Tensor cache, Tensor block_table,
                   OptTensor row_item, Tensor row_len, Tensor sink,
                   long window, double scale) {
  CHK_DEV(qa); CHK_CONT(qa); CHK_CONT(cache); CHK_SAME(qa, cache);
  CHK_SAME(qa, sink); CHK_CONT(sink); CHK_I32(block_table); CHK_I32(row_len);
  const int R = (int)qa.size(0), H = (int)sink.numel();
  TORCH_CHECK(cache.dim() == 3 && cache.size(1) == 64, "cache [P, 64, KR]");
  const int KR = (int)cache.size(2);
  TORCH_CHECK(qa.dim() == 2 && qa.size(1) == (long long)H * KR, "qa [R, H*KR]");
  TORCH_CHECK(row_len.numel() == R && block_table.dim() == 2, "row arrays");
  TORCH_CHECK(KR <= 8000, "latent too wide");
  const int* ri = nullptr;
  if (row_item) {
    CHK_I32(*row_item);
    TORCH_CHECK(row_item->numel() == R, "row_item");
    ri = row_item->data_ptr<int>();
  } else {
    TORCH_CHECK(block_table.size(0) >= R, "block_table rows");
  }
  auto out = torch::empty_like(qa);
  if (R == 0) return out;
  const int mp = (int)block_table.size(1);
  const int f32 = is_f32(qa);
  if (!f32 && KR % 8 == 0 && KR <= 512) {
    const int HT = (H + 15) / 16;
    int pages = mp;
    if (window > 0) pages = (int)std::min<long>(mp, (window + 62) / 64 + 1);
    // two blocks fit a CU: enough of them to fill the chip once, and no
    // shares that differ by a page when they need not
    long long ns = (512 + (long long)R * HT - 1) / ((long long)R * HT);
    ns = std::max<long long>(1, std::min<long long>(ns, pages));
    const long long per = (pages + ns - 1) / ns;
    ns = (pages + per - 1) / per;
    auto of = qa.options().dtype(at::kFloat);
    auto po = torch::empty({R, H, ns, KR}, of);
    auto pm = torch::empty({R, H, ns, 2}, of);
    qsa_latent_rows_mfma_launch(
        u16(qa), u16(cache), block_table.data_ptr<int>(), mp, ri,
        row_len.data_ptr<int>(), u16(sink), po.data_ptr<float>(),
        pm.data_ptr<float>(), u16m(out), R, H, KR, (int)window, (float)scale,
        (int)ns, cur_stream());
  } else {
    qsa_latent_rows_launch(qa.data_ptr(), cache.data_ptr(),
                           block_table.data_ptr<int>(), mp, ri,
                           row_len.data_ptr<int>(), sink.data_ptr(),
                           out.data_ptr(), R, H, KR, (int)window,
                           (float)scale, f32, cur_stream());
  }
  return out;
}

bool window_attn_ok(long H, long D, long E) {
  return D <= 256 && E <= 256 && D % 8 == 0 && E % 8 == 0;
}

// portions' rows of q [T, H*D] against expanded context kv [C, H*(D+E)];
// writes sigmoid(gate) * attention into the same rows of out [T, H*E]
void window_attn_prefill(Tensor q, Tensor kv, Tensor gate, Tensor sink,
                         Tensor qb_item, Tensor qb_t0, Tensor off,
                         Tensor start, Tensor len, Tensor ctx_off,
                         Tensor ctx_pos, Tensor out, long D, long E,
                         long window, double scale) {
  CHK_DEV(q); chk_rows(q, "q"); chk_rows(kv, "kv"); chk_rows(gate, "gate");
  CHK_CONT(out); CHK_CONT(sink);
  TORCH_CHECK(q.scalar_type() == at::kBFloat16, "bf16 storage");
  CHK_SAME(q, kv); CHK_SAME(q, gate); CHK_SAME(q, sink); CHK_SAME(q, out);
  CHK_I32(qb_item); CHK_I32(qb_t0); CHK_I32(off); CHK_I32(start);
  CHK_I32(len); CHK_I32(ctx_off); CHK_I32(ctx_pos);
  const int H = (int)sink.numel();
  TORCH_CHECK(window_attn_ok(H, D, E), "head sizes of the matrix-core path");
  TORCH_CHECK(q.size(1) == H * D && kv.size(1) == H * (D + E) &&
                  gate.size(1) == H * E && out.size(1) == H * E &&
                  gate.size(0) == q.size(0) && out.size(0) == q.size(0),
              "operand shapes");
  TORCH_CHECK(q.stride(0) % 8 == 0 && kv.stride(0) % 8 == 0 &&
                  gate.stride(0) % 4 == 0 && aligned(q, 16) &&
                  aligned(kv, 16) && aligned(gate, 8), "alignment");
  const int QB = (int)qb_item.numel();
  const auto n = off.numel();
  TORCH_CHECK(qb_t0.numel() == QB && start.numel() == n && len.numel() == n &&
                  ctx_off.numel() == n && ctx_pos.numel() == n, "plan arrays");
  if (QB == 0) return;
  qsa_window_attn_prefill_launch(
      u16(q), q.stride(0), u16(kv), kv.stride(0), u16(gate), gate.stride(0),
      u16(sink), qb_item.data_ptr<int>(), qb_t0.data_ptr<int>(),
      off.data_ptr<int>(), start.data_ptr<int>(), len.data_ptr<int>(),
      ctx_off.data_ptr<int>(), ctx_pos.data_ptr<int>(), u16m(out), QB, H,
      (int)D, (int)E, (int)window, (float)scale, cur_stream());
}

// ---- short convolutions ----------------------------------------------------
// Portions with chunks of 16 rows (item, t0), or, without `item`, one token
// per row at position start - 1.
static int conv_step(ConvStep& st, const OptTensor& item, const OptTensor& t0,
                     const OptTensor& off, const Tensor& start,
                     const OptTensor& len, const Tensor& slots, long rows) {
  CHK_I32(start); CHK_I32(slots);
  TORCH_CHECK(start.numel() == slots.numel(), "one slot per portion");
  st = ConvStep{nullptr, nullptr, nullptr, start.data_ptr<int>(), nullptr,
                slots.data_ptr<int>()};
  if (!item) {
    TORCH_CHECK(start.numel() == rows, "one row per sequence");
    return (int)rows;
  }
  TORCH_CHECK(t0 && off && len, "portions need t0, off and len");
  CHK_I32(*item); CHK_I32(*t0); CHK_I32(*off); CHK_I32(*len);
  TORCH_CHECK(t0->numel() == item->numel() &&
                  off->numel() == start.numel() &&
                  len->numel() == start.numel(), "per-portion arrays");
  st.item = item->data_ptr<int>(); st.t0 = t0->data_ptr<int>();
  st.off = off->data_ptr<int>(); st.len = len->data_ptr<int>();
  return (int)item->numel();
}

static void chk_conv(const Tensor& x, const Tensor& w, const Tensor& tails,
                     long C) {
  CHK_DEV(x); chk_rows(x, "x"); CHK_F32(w); CHK_CONT(tails);
  CHK_SAME(x, tails);
  TORCH_CHECK(w.dim() == 2 && w.size(1) == C, "filters [taps, C]");
  TORCH_CHECK(w.size(0) >= 1 && w.size(0) <= 17, "1 to 17 taps");
  TORCH_CHECK(tails.dim() == 3 && tails.size(1) == w.size(0) - 1 &&
                  tails.size(2) == C, "tails [slots, taps - 1, C]");
  TORCH_CHECK(x.size(1) >= C, "columns");
}

// x columns [q | k | v]; returns rotated q [T, H*D], k and v to their pages
Tensor conv_qkv(Tensor x, Tensor w, Tensor tails, Tensor cos_t, Tensor sin_t,
                long rot, Tensor cache_slots, Tensor kc, Tensor vc, long H,
                OptTensor item, OptTensor t0, OptTensor off, Tensor start,
                OptTensor len, Tensor slots) {
  CHK_CONT(kc); CHK_CONT(vc); CHK_SAME(x, kc); CHK_SAME(x, vc);
  CHK_I32(cache_slots);
  TORCH_CHECK(kc.dim() == 4 && kc.size(2) == 64 && vc.dim() == 4 &&
                  vc.size(2) == 64 && vc.size(0) == kc.size(0) &&
                  vc.size(1) == kc.size(1), "pages [P, G, 64, D], [P, G, 64, E]");
  const int G = (int)kc.size(1), D = (int)kc.size(3), E = (int)vc.size(3);
  const long C = (H + G) * (long)D + (long)G * E;
  chk_conv(x, w, tails, C);
  TORCH_CHECK(rot % 2 == 0 && rot >= 0 && rot <= D, "rotated dims");
  int table_len = 0x7fffffff;
  if (rot > 0) {
    CHK_F32(cos_t); CHK_F32(sin_t);
    TORCH_CHECK(cos_t.dim() == 2 && cos_t.size(1) == rot / 2 &&
                    sin_t.sizes() == cos_t.sizes() && cos_t.size(0) > 0,
                "rotation tables");
    table_len = (int)cos_t.size(0);
  }
  const long T = x.size(0);
  TORCH_CHECK(cache_slots.numel() == T, "one cache slot per row");
  auto q = torch::empty({T, H * (long)D}, x.options());
  if (T == 0) return q;
  ConvStep st;
  const int chunks = conv_step(st, item, t0, off, start, len, slots, T);
  const int v4 = D % 4 == 0 && E % 4 == 0 && rot % 8 == 0 &&
                 x.stride(0) % 4 == 0 && aligned(x, is_f32(x) ? 16 : 8);
  qsa_conv_qkv_launch(x.data_ptr(), x.stride(0), w.data_ptr<float>(),
                      (int)w.size(0), tails.data_ptr(), st, chunks,
                      rot ? cos_t.data_ptr<float>() : nullptr,
                      rot ? sin_t.data_ptr<float>() : nullptr, (int)rot,
                      table_len, cache_slots.data_ptr<int>(), q.data_ptr(),
                      kc.data_ptr(), vc.data_ptr(), (int)H, G, D, E,
                      is_f32(x), v4, cur_stream());
  return q;
}

// silu(conv(x) + bias) -> dense [T, C]
Tensor conv_silu(Tensor x, Tensor w, Tensor bias, Tensor tails,
                 OptTensor item, OptTensor t0, OptTensor off, Tensor start,
                 OptTensor len, Tensor slots) {
  const long T = x.size(0), C = x.size(1);
  chk_conv(x, w, tails, C);
  CHK_F32(bias);
  TORCH_CHECK(bias.numel() == C, "bias");
  auto out = torch::empty({T, C}, x.options());
  if (T == 0) return out;
  ConvStep st;
  const int chunks = conv_step(st, item, t0, off, start, len, slots, T);
  const int v4 = C % 4 == 0 && x.stride(0) % 4 == 0 &&
                 aligned(x, is_f32(x) ? 16 : 8);
  qsa_conv_silu_launch(x.data_ptr(), x.stride(0), w.data_ptr<float>(),
                       bias.data_ptr<float>(), (int)w.size(0),
                       tails.data_ptr(), st, chunks, out.data_ptr(), (int)C,
                       is_f32(x), v4, cur_stream());
  return out;
}

// ---- grouped-query attention over pages ------------------------------------
struct GqaDims { int R, H, G, D, E; };

static GqaDims gqa_check(const Tensor& q, const Tensor& kc, const Tensor& vc,
                         const Tensor& block_table, const OptTensor& sink,
                         const OptTensor& gate, const Tensor& out, long H) {
  CHK_DEV(q); CHK_CONT(q); CHK_CONT(kc); CHK_CONT(vc); CHK_SAME(q, kc);
  CHK_SAME(q, vc); CHK_SAME(q, out); chk_rows(out, "out");
  CHK_I32(block_table);
  TORCH_CHECK(block_table.dim() == 2, "block_table [items, pages]");
  TORCH_CHECK(kc.dim() == 4 && kc.size(2) == 64 && vc.dim() == 4 &&
                  vc.size(2) == 64 && vc.size(0) == kc.size(0) &&
                  vc.size(1) == kc.size(1), "pages [P, G, 64, D], [P, G, 64, E]");
  GqaDims d{(int)q.size(0), (int)H, (int)kc.size(1), (int)kc.size(3),
            (int)vc.size(3)};
  TORCH_CHECK(q.dim() == 2 && q.size(1) == H * d.D, "q [R, H*D]");
  TORCH_CHECK(d.G > 0 && H % d.G == 0, "query heads per key head");
  TORCH_CHECK(out.size(0) == d.R && out.size(1) == H * d.E, "out [R, H*E]");
  if (sink) {
    CHK_F32(*sink);
    TORCH_CHECK(sink->numel() == H, "one sink per head");
  }
  if (gate) {
    CHK_SAME(q, *gate); chk_rows(*gate, "gate");
    TORCH_CHECK(gate->size(0) == d.R && gate->size(1) == H * d.E, "gate");
  }
  return d;
}

bool gqa_mfma_ok(long D, long E) {
  return D <= 256 && E <= 256 && D % 8 == 0 && E % 8 == 0;
}

static bool gqa_aligned(const Tensor& q, const OptTensor& gate,
                        const Tensor& out) {
  return aligned(q, 16) && out.stride(0) % 4 == 0 && aligned(out, 8) &&
         (!gate || (gate->stride(0) % 4 == 0 && aligned(*gate, 8)));
}

// q [R, H*D] rows -> rows of out; row_item: which block_table row a query row
// uses (none: its own index); row_len: position + 1 (0: row not in use)
void gqa_rows(Tensor q, Tensor kc, Tensor vc, Tensor block_table,
              OptTensor row_item, Tensor row_len, OptTensor sink,
              OptTensor gate, Tensor out, long H, double scale,
              double out_scale) {
  const GqaDims d = gqa_check(q, kc, vc, block_table, sink, gate, out, H);
  CHK_I32(row_len);
  TORCH_CHECK(row_len.numel() == d.R, "row arrays");
  const int* ri = nullptr;
  if (row_item) {
    CHK_I32(*row_item);
    TORCH_CHECK(row_item->numel() == d.R, "row_item");
    ri = row_item->data_ptr<int>();
  } else {
    TORCH_CHECK(block_table.size(0) >= d.R, "block_table rows");
  }
  if (d.R == 0) return;
  const int mp = (int)block_table.size(1);
  const int f32 = is_f32(q);
  const float* sp = sink ? sink->data_ptr<float>() : nullptr;
  const void* gp = gate ? gate->data_ptr() : nullptr;
  const long long gs = gate ? gate->stride(0) : 0;
  if (!f32 && gqa_mfma_ok(d.D, d.E) && gqa_aligned(q, gate, out)) {
    // two waves a SIMD fill the chip; no shares that differ by a page when
    // they need not
    const long long tiles =
        (long long)d.R * d.G * ((d.H / d.G + 15) / 16);
    long long ns = (2048 + tiles - 1) / tiles;
    ns = std::max<long long>(1, std::min<long long>(ns, mp));
    const long long per = (mp + ns - 1) / ns;
    ns = (mp + per - 1) / per;
    TORCH_CHECK(tiles * ns < (1LL << 31), "rows per call");
    auto of = q.options().dtype(at::kFloat);
    auto po = torch::empty({d.R, d.H, ns, d.E}, of);
    auto pm = torch::empty({d.R, d.H, ns, 2}, of);
    qsa_gqa_rows_mfma_launch(
        u16(q), u16(kc), u16(vc), block_table.data_ptr<int>(), mp, ri,
        row_len.data_ptr<int>(), sp, (const bf16_t*)gp, gs,
        po.data_ptr<float>(), pm.data_ptr<float>(), u16m(out), out.stride(0),
        d.R, d.H, d.G, d.D, d.E, (float)scale, (float)out_scale, (int)ns,
        cur_stream());
  } else {
    TORCH_CHECK(d.D + d.E <= 12000, "head too wide");
    qsa_gqa_rows_launch(q.data_ptr(), kc.data_ptr(), vc.data_ptr(),
                        block_table.data_ptr<int>(), mp, ri,
                        row_len.data_ptr<int>(), sp, gp, gs, out.data_ptr(),
                        out.stride(0), d.R, d.H, d.G, d.D, d.E, (float)scale,
                        (float)out_scale, f32, cur_stream());
  }
}

// query rows a block of gqa_portions takes
long gqa_portion_rows(long D, long E) {
  return D <= 128 && E <= 128 ? 128 : 64;
}

// portions' rows of q; block_table row i belongs to portion i
void gqa_portions(Tensor q, Tensor kc, Tensor vc, Tensor block_table,
                  OptTensor sink, OptTensor gate, Tensor qb_item,
                  Tensor qb_t0, Tensor off, Tensor start, Tensor len,
                  Tensor out, long H, double scale, double out_scale) {
  const GqaDims d = gqa_check(q, kc, vc, block_table, sink, gate, out, H);
  TORCH_CHECK(q.scalar_type() == at::kBFloat16, "bf16 storage");
  TORCH_CHECK(gqa_mfma_ok(d.D, d.E) && gqa_aligned(q, gate, out),
              "head sizes and alignment of the matrix-core path");
  CHK_I32(qb_item); CHK_I32(qb_t0); CHK_I32(off); CHK_I32(start);
  CHK_I32(len);
  const int QB = (int)qb_item.numel();
  const auto n = off.numel();
  TORCH_CHECK(qb_t0.numel() == QB && start.numel() == n && len.numel() == n &&
                  block_table.size(0) == n, "plan arrays");
  if (QB == 0) return;
  qsa_gqa_portions_launch(
      u16(q), u16(kc), u16(vc), block_table.data_ptr<int>(),
      (int)block_table.size(1), sink ? sink->data_ptr<float>() : nullptr,
      gate ? u16(*gate) : nullptr, gate ? gate->stride(0) : 0,
      qb_item.data_ptr<int>(), qb_t0.data_ptr<int>(), off.data_ptr<int>(),
      start.data_ptr<int>(), len.data_ptr<int>(), u16m(out), out.stride(0),
      QB, d.H, d.G, d.D, d.E, (float)scale, (float)out_scale,
      gqa_portion_rows(d.D, d.E) == 128, cur_stream());
}

// ---- state-space duality ---------------------------------------------------
struct SsdDims { int H, N, P, G; };

static SsdDims ssd_check(const Tensor& u, const Tensor& xbc, const Tensor& A,
                         const Tensor& dt_bias, const Tensor& D,
                         const Tensor& state, const Tensor& out, long G,
                         long zoff, long dtoff) {
  CHK_DEV(u); chk_rows(u, "u"); CHK_CONT(xbc); CHK_CONT(out);
  CHK_SAME(u, xbc); CHK_SAME(u, out); CHK_F32(A); CHK_F32(dt_bias);
  CHK_F32(D); CHK_F32(state);
  TORCH_CHECK(state.dim() == 4, "state [slots, H, N, P]");
  SsdDims s{(int)state.size(1), (int)state.size(2), (int)state.size(3),
            (int)G};
  const long inner = (long)s.H * s.P;
  TORCH_CHECK(G > 0 && s.H % G == 0, "heads per group");
  TORCH_CHECK(A.numel() == s.H && dt_bias.numel() == s.H &&
                  D.numel() == s.H, "per-head constants");
  TORCH_CHECK(xbc.dim() == 2 && xbc.size(0) == u.size(0) &&
                  xbc.size(1) == inner + 2 * G * s.N, "xbc [T, x | B | C]");
  TORCH_CHECK(out.dim() == 2 && out.size(0) == u.size(0) &&
                  out.size(1) == inner, "out [T, H*P]");
  TORCH_CHECK(zoff >= 0 && zoff + inner <= u.size(1) && dtoff >= 0 &&
                  dtoff + s.H <= u.size(1), "columns of z and dt");
  return s;
}

Tensor ssd_decode(Tensor u, long zoff, long dtoff, Tensor xbc, Tensor A,
                  Tensor dt_bias, Tensor D, Tensor state, long G,
                  Tensor slots, Tensor seq_lens) {
  auto out = torch::empty({u.size(0), state.size(1) * state.size(3)},
                          u.options());
  const SsdDims s = ssd_check(u, xbc, A, dt_bias, D, state, out, G, zoff,
                              dtoff);
  CHK_I32(slots); CHK_I32(seq_lens);
  const int B = (int)u.size(0);
  TORCH_CHECK(slots.numel() == B && seq_lens.numel() == B, "slots/seq_lens");
  TORCH_CHECK(s.N <= 5000, "state too wide for the decode block");
  if (B == 0) return out;
  const int a = is_f32(u) ? 16 : 8;
  const int v4 = s.P % 4 == 0 && xbc.size(1) % 4 == 0 && zoff % 4 == 0 &&
                 u.stride(0) % 4 == 0 && aligned(u, a) && aligned(xbc, a);
  qsa_ssd_decode_launch(
      u.data_ptr(), u.stride(0), (int)zoff, (int)dtoff, xbc.data_ptr(),
      A.data_ptr<float>(), dt_bias.data_ptr<float>(), D.data_ptr<float>(),
      state.data_ptr<float>(), slots.data_ptr<int>(),
      seq_lens.data_ptr<int>(), out.data_ptr(), B, s.H, s.N, s.P, s.G,
      is_f32(u), v4, cur_stream());
  return out;
}

void ssd_seq(Tensor u, long zoff, long dtoff, Tensor xbc, Tensor A,
             Tensor dt_bias, Tensor D, Tensor state, long G, Tensor slots,
             Tensor off, Tensor start, Tensor len, Tensor out) {
  const SsdDims s = ssd_check(u, xbc, A, dt_bias, D, state, out, G, zoff,
                              dtoff);
  const int n = chk_items(slots, off, start, len);
  TORCH_CHECK(s.N <= 5000, "state too wide");
  if (n == 0) return;
  qsa_ssd_seq_launch(
      u.data_ptr(), u.stride(0), (int)zoff, (int)dtoff, xbc.data_ptr(),
      A.data_ptr<float>(), dt_bias.data_ptr<float>(), D.data_ptr<float>(),
      state.data_ptr<float>(), slots.data_ptr<int>(), off.data_ptr<int>(),
      start.data_ptr<int>(), len.data_ptr<int>(), out.data_ptr(), n, s.H,
      s.N, s.P, s.G, is_f32(u), cur_stream());
}

bool ssd_chunked_ok(long H, long N, long P, long G) {
  return N <= 256 && P <= 256 && N % 8 == 0 && P % 8 == 0 && H % G == 0;
}

// chunked prefill of the portions (chunks of 64 tokens)
void ssd_chunked(Tensor u, long zoff, long dtoff, Tensor xbc, Tensor A,
                 Tensor dt_bias, Tensor D, Tensor state, long G, Tensor slots,
                 Tensor off, Tensor start, Tensor len, Tensor chunk0,
                 Tensor chunk_item, Tensor chunk_t0, Tensor out) {
  const SsdDims s = ssd_check(u, xbc, A, dt_bias, D, state, out, G, zoff,
                              dtoff);
  const int n = chk_items(slots, off, start, len);
  CHK_I32(chunk0); CHK_I32(chunk_item); CHK_I32(chunk_t0);
  TORCH_CHECK(u.scalar_type() == at::kBFloat16, "bf16 storage");
  TORCH_CHECK(ssd_chunked_ok(s.H, s.N, s.P, G), "sizes of the chunked path");
  TORCH_CHECK(zoff % 4 == 0 && u.stride(0) % 4 == 0 && aligned(u, 8) &&
                  aligned(xbc, 16), "alignment");
  const long long nc = chunk_item.numel();
  TORCH_CHECK(chunk0.numel() == n && chunk_t0.numel() == nc, "plan arrays");
  if (n == 0 || nc == 0) return;
  const int DP = pad_dim(s.N), EP = (s.P + 15) / 16 * 16;
  auto steps = torch::empty({nc, s.H, 2, 64}, u.options().dtype(at::kFloat));
  auto prefix = torch::empty({nc, s.H, 2, EP, DP}, u.options());
  hipStream_t st = cur_stream();
  qsa_ssd_steps_launch(u16(u), u.stride(0), (int)dtoff, A.data_ptr<float>(),
                       dt_bias.data_ptr<float>(), off.data_ptr<int>(),
                       len.data_ptr<int>(), chunk_item.data_ptr<int>(),
                       chunk_t0.data_ptr<int>(), steps.data_ptr<float>(),
                       (int)nc, s.H, st);
  qsa_ssd_state_launch(u16(xbc), steps.data_ptr<float>(),
                       state.data_ptr<float>(), slots.data_ptr<int>(),
                       off.data_ptr<int>(), start.data_ptr<int>(),
                       len.data_ptr<int>(), chunk0.data_ptr<int>(),
                       prefix.data_ptr(), n, s.H, s.N, DP, s.P, EP, s.G, st);
  qsa_ssd_out_launch(u16(u), u.stride(0), (int)zoff, u16(xbc),
                     steps.data_ptr<float>(), D.data_ptr<float>(),
                     off.data_ptr<int>(), start.data_ptr<int>(),
                     len.data_ptr<int>(), chunk_item.data_ptr<int>(),
                     chunk_t0.data_ptr<int>(), prefix.data_ptr(), (int)nc,
                     u16m(out), s.H, s.N, DP, s.P, EP, s.G, st);
}

// rms norm of `parts` equal parts of a row, times w -> rows of out
void part_norm(Tensor x, Tensor w, Tensor out, long parts, double eps) {
  CHK_DEV(x); CHK_CONT(x); CHK_F32(w); CHK_SAME(x, out);
  chk_rows(out, "out");
  TORCH_CHECK(x.dim() == 2 && out.sizes() == x.sizes() &&
                  w.numel() == x.size(1), "x, w, out shapes");
  TORCH_CHECK(parts > 0 && x.size(1) % parts == 0, "equal parts");
  const int n = (int)(x.size(1) / parts);
  if (x.numel() == 0) return;
  const int a = is_f32(x) ? 16 : 8;
  const int v = n % 4 == 0 && out.stride(0) % 4 == 0 && aligned(x, a) &&
                aligned(out, a);
  qsa_part_norm_launch(x.data_ptr(), w.data_ptr<float>(), out.data_ptr(),
                       out.stride(0), x.size(0), (int)parts, n, (float)eps,
                       is_f32(x), v, cur_stream());
}

// weight-streaming decode product, W packed as [N/16, K/32, 16, 32]
Tensor skinny_gemm(Tensor a, Tensor wf, long N, long K) {
  CHK_DEV(a); chk_rows(a, "a"); CHK_CONT(wf); CHK_SAME(a, wf);
  TORCH_CHECK(a.scalar_type() == at::kBFloat16, "bf16");
  const int M = (int)a.size(0);
  TORCH_CHECK(M >= 1 && M <= 32 && a.size(1) == K, "M in [1, 32], K");
  TORCH_CHECK(K % 256 == 0 && N % 16 == 0 && wf.numel() == N * K, "W packing");
  TORCH_CHECK(a.stride(0) % 8 == 0 && aligned(a, 16), "a alignment");
  auto out = torch::empty({M, (long long)N}, a.options());
  qsa_skinny_gemm_launch(u16(a), u16(wf), u16m(out), M, (int)N, K,
                         a.stride(0), cur_stream());
  return out;
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("residual_norm", &residual_norm,
        "f32 residual update (+ embedding row, + vector) and layer/rms norm");
  m.def("glu", &glu, "act(gate) * up, bf16 or f32, any size");
  m.def("glu_table", &glu_table, "act(gate) * slice of the token's table row");
  m.def("conv_qkv", &conv_qkv,
        "short convolutions of q, k, v; rotation; k, v to their pages");
  m.def("conv_silu", &conv_silu, "short convolution with bias and silu");
  m.def("gqa_rows", &gqa_rows, "paged grouped-query attention of rows");
  m.def("gqa_portions", &gqa_portions,
        "paged grouped-query flash attention with sink and gate (MFMA)");
  m.def("gqa_mfma_ok", &gqa_mfma_ok, "size support");
  m.def("gqa_portion_rows", &gqa_portion_rows, "query rows per block");
  m.def("ssd_decode", &ssd_decode, "one token per row");
  m.def("ssd_seq", &ssd_seq, "token loop over portions");
  m.def("ssd_chunked", &ssd_chunked, "chunked prefill (MFMA)");
  m.def("ssd_chunked_ok", &ssd_chunked_ok, "size support");
  m.def("part_norm", &part_norm, "rms norm in equal parts of a row");
  m.def("latent_norm_store", &latent_norm_store,
        "rms norms of the query and kv latents; kv latent to the cache");
  m.def("decode_slots", &decode_slots, "cache slot of each row's new position");
  m.def("argmax_rows", &argmax_rows, "greedy pick per row");
  m.def("retention_decode", &retention_decode, "one token per row");
  m.def("retention_seq", &retention_seq, "token loop over portions");
  m.def("retention_chunked", &retention_chunked, "chunked prefill (MFMA)");
  m.def("retention_chunked_ok", &retention_chunked_ok, "size support");
  m.def("head_matmul", &head_matmul, "per-head product (+ sigmoid gate)");
  m.def("latent_rows", &latent_rows, "absorbed latent attention of rows");
  m.def("window_attn_prefill", &window_attn_prefill,
        "windowed flash attention with sink and gate (MFMA)");
  m.def("window_attn_ok", &window_attn_ok, "size support");
  m.def("skinny_gemm", &skinny_gemm, "packed-weight decode GEMM (M <= 32)");
}
