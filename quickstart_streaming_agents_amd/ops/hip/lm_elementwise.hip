// Row kernels of the mixer decoders: residual update + norm in f32, gated
// activation, latent norm + cache scatter, step slots, greedy pick.
#include "lm_common.h"

// ---------------------------------------------------------------------------
// Residual update and norm of one row, everything in f32:
//   r   = (init ? 0 : res) + p + tscale * table[ids[row]] + vec
//         (p, table, vec optional); p = y, or with POST the branch's own norm
//         y / sqrt(mean y^2 + eps) * post
//   res = r
//   out = norm(r) * w + b      LAYER: (r - mean)/sqrt(var + eps), var the
//                              mean squared deviation; else r/sqrt(mean r^2
//                              + eps).  b optional; without w, out = r.
// The row stays in registers between the passes up to CACHED groups per
// thread; wider rows re-read the residual this thread wrote itself.
// ---------------------------------------------------------------------------
template <typename T, int VEC, bool LAYER, bool POST>
__global__ void __launch_bounds__(1024)
qsa_residual_norm(float* __restrict__ res, const T* __restrict__ y,
                  long long ystride, const T* __restrict__ post,
                  const T* __restrict__ table,
                  const long long* __restrict__ ids, float tscale,
                  const T* __restrict__ vec, const T* __restrict__ w,
                  const T* __restrict__ b, T* __restrict__ out, int W,
                  int vocab, float eps, int init) {
  constexpr int CACHED = 8;
  __shared__ float scratch[16];
  const long long row = blockIdx.x;
  float* rr = res + row * W;
  const T* yr = y ? y + row * ystride : nullptr;
  const T* er = nullptr;
  if (table) {
    long long id = ids[row];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
    er = table + id * W;
  }
  const int step = blockDim.x * VEC;
  const int i0 = threadIdx.x * VEC;
  float cache[CACHED][VEC];
  float pinv = 1.f;
  if (POST) {
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < CACHED; ++c) {
      const int i = i0 + c * step;
      if (i < W) {
        ldv<T, VEC>(yr + i, cache[c]);
#pragma unroll
        for (int j = 0; j < VEC; ++j) ss = fmaf(cache[c][j], cache[c][j], ss);
      }
    }
    for (int i = i0 + CACHED * step; i < W; i += step) {
      float v[VEC];
      ldv<T, VEC>(yr + i, v);
#pragma unroll
      for (int j = 0; j < VEC; ++j) ss = fmaf(v[j], v[j], ss);
    }
    pinv = 1.f / sqrtf(block_reduce_sum(ss, scratch) / (float)W + eps);
  }
  float sum = 0.f;
  // v: on entry, with POST, the branch's output
  auto load_row = [&](int i, float* v) {
    float t[VEC];
    if (POST) {
      ldv<T, VEC>(post + i, t);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] *= pinv * t[j];
      if (!init) {
        ldv<float, VEC>(rr + i, t);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] += t[j];
      }
    } else {
      if (init) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] = 0.f;
      } else {
        ldv<float, VEC>(rr + i, v);
      }
      if (yr) {
        ldv<T, VEC>(yr + i, t);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] += t[j];
      }
    }
    if (er) {
      ldv<T, VEC>(er + i, t);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = fmaf(tscale, t[j], v[j]);
    }
    if (vec) {
      ldv<T, VEC>(vec + i, t);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] += t[j];
    }
    stv<float, VEC>(rr + i, v);
  };
#pragma unroll
  for (int c = 0; c < CACHED; ++c) {
    const int i = i0 + c * step;
    if (i < W) {
      load_row(i, cache[c]);
#pragma unroll
      for (int j = 0; j < VEC; ++j)
        sum += LAYER ? cache[c][j] : cache[c][j] * cache[c][j];
    }
  }
  for (int i = i0 + CACHED * step; i < W; i += step) {
    float v[VEC];
    if (POST) ldv<T, VEC>(yr + i, v);
    load_row(i, v);
#pragma unroll
    for (int j = 0; j < VEC; ++j) sum += LAYER ? v[j] : v[j] * v[j];
  }
  T* orow = out + row * W;
  if (!w) {                                         // the residual itself
#pragma unroll
    for (int c = 0; c < CACHED; ++c)
      if (i0 + c * step < W) stv<T, VEC>(orow + i0 + c * step, cache[c]);
    for (int i = i0 + CACHED * step; i < W; i += step) {
      float v[VEC];
      ldv<float, VEC>(rr + i, v);
      stv<T, VEC>(orow + i, v);
    }
    return;
  }
  sum = block_reduce_sum(sum, scratch);
  float mean = 0.f, ms = sum / (float)W;
  if (LAYER) {
    mean = ms;
    float dev = 0.f;
#pragma unroll
    for (int c = 0; c < CACHED; ++c)
      if (i0 + c * step < W) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          const float d = cache[c][j] - mean;
          dev = fmaf(d, d, dev);
        }
      }
    for (int i = i0 + CACHED * step; i < W; i += step) {
      float v[VEC];
      ldv<float, VEC>(rr + i, v);
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        const float d = v[j] - mean;
        dev = fmaf(d, d, dev);
      }
    }
    ms = block_reduce_sum(dev, scratch) / (float)W;
  }
  const float inv = 1.f / sqrtf(ms + eps);
  auto emit = [&](int i, const float* v) {
    float t[VEC], o[VEC];
    ldv<T, VEC>(w + i, t);
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = (v[j] - mean) * inv * t[j];
    if (b) {
      ldv<T, VEC>(b + i, t);
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] += t[j];
    }
    stv<T, VEC>(orow + i, o);
  };
#pragma unroll
  for (int c = 0; c < CACHED; ++c)
    if (i0 + c * step < W) emit(i0 + c * step, cache[c]);
  for (int i = i0 + CACHED * step; i < W; i += step) {
    float v[VEC];
    ldv<float, VEC>(rr + i, v);
    emit(i, v);
  }
}

template <typename T, int VEC, bool LAYER, bool POST>
static void residual_norm_go(float* res, const void* y, long long ystride,
                             const void* post, const void* table,
                             const long long* ids, float tscale,
                             const void* vec, const void* w, const void* b,
                             void* out, long long rows, int W, int vocab,
                             float eps, int init, hipStream_t st) {
  int threads = ((W + VEC - 1) / VEC + 63) / 64 * 64;
  // few rows: wide blocks, one round of loads; many rows: narrow ones
  const int most = rows <= 256 ? 1024 : 256;
  threads = threads > most ? most : threads;
  hipLaunchKernelGGL((qsa_residual_norm<T, VEC, LAYER, POST>),
                     dim3((unsigned)rows), dim3(threads), 0, st, res,
                     (const T*)y, ystride, (const T*)post, (const T*)table,
                     ids, tscale, (const T*)vec, (const T*)w, (const T*)b,
                     (T*)out, W, vocab, eps, init);
}

extern "C" void qsa_residual_norm_launch(
    float* res, const void* y, long long ystride, const void* post,
    const void* table, const long long* ids, float tscale, const void* vec,
    const void* w, const void* b, void* out, long long rows, int W, int vocab,
    float eps, int init, int layer, int f32, int vec4, hipStream_t st) {
#define QSA_RN(T, V, L, P)                                                    \
  residual_norm_go<T, V, L, P>(res, y, ystride, post, table, ids, tscale,     \
                               vec, w, b, out, rows, W, vocab, eps, init, st)
#define QSA_RN_L(T, V)                                                        \
  if (layer) { if (post) QSA_RN(T, V, true, true);                            \
               else QSA_RN(T, V, true, false); }                              \
  else { if (post) QSA_RN(T, V, false, true);                                 \
         else QSA_RN(T, V, false, false); }
  if (f32) {
    if (vec4) { QSA_RN_L(float, 4) } else { QSA_RN_L(float, 1) }
  } else {
    if (vec4) { QSA_RN_L(bf16_t, 4) } else { QSA_RN_L(bf16_t, 1) }
  }
#undef QSA_RN_L
#undef QSA_RN
}

// ---------------------------------------------------------------------------
// Gated activations.  The factor is the other half of a projection (a gated
// linear unit) or a slice of the token's row of a table:
//   out[r, c] = act(gate[r, c]) * up[r, c]
//   out[r, c] = act(gate[r, c]) * table[ids[r], col0 + c]
// act: silu, or the tanh form of gelu, z / (1 + exp(-2 sqrt(2/pi)
// (z + 0.044715 z^3))).
// ---------------------------------------------------------------------------
#define QSA_ACT_SILU 0
#define QSA_ACT_GELU 1

template <bool EXACT, int ACT>
__device__ __forceinline__ float act_f(float z) {
  const float a = ACT == QSA_ACT_SILU
      ? z : 1.5957691216057308f * fmaf(0.044715f * z * z, z, z);
  return z / (1.f + (EXACT ? expf(-a) : __expf(-a)));
}

template <typename T, int VEC, int ACT>
__global__ void __launch_bounds__(256)
qsa_glu(const T* __restrict__ gate, const T* __restrict__ up,
        const long long* __restrict__ ids, T* __restrict__ out,
        long long rows, long long cols, long long stride, long long ustride,
        long long vocab) {
  const long long groups = cols / VEC;
  const long long n = rows * groups;
  for (long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x; i < n;
       i += (long long)gridDim.x * blockDim.x) {
    const long long r = i / groups, c = (i % groups) * VEC;
    long long ur = r;
    if (ids) {
      ur = ids[r];
      ur = ur < 0 ? 0 : (ur >= vocab ? vocab - 1 : ur);
    }
    float g[VEC], u[VEC];
    ldv<T, VEC>(gate + r * stride + c, g);
    ldv<T, VEC>(up + ur * ustride + c, u);
#pragma unroll
    for (int j = 0; j < VEC; ++j)
      g[j] = act_f<sizeof(T) == 4, ACT>(g[j]) * u[j];
    stv<T, VEC>(out + r * cols + c, g);
  }
}

extern "C" void qsa_glu_launch(const void* gate, const void* up,
                               const long long* ids, void* out,
                               long long rows, long long cols,
                               long long stride, long long ustride,
                               long long vocab, int gelu, int f32, int vec,
                               hipStream_t st) {
  const long long n = rows * (cols / (vec ? 8 : 1));
  const long long want = (n + 255) / 256;
  dim3 grid((unsigned)(want < 1 ? 1 : (want > 16384 ? 16384 : want)));
#define QSA_GLU(T, V, A)                                                   \
  hipLaunchKernelGGL((qsa_glu<T, V, A>), grid, dim3(256), 0, st,           \
                     (const T*)gate, (const T*)up, ids, (T*)out, rows,     \
                     cols, stride, ustride, vocab)
#define QSA_GLU_A(T, V)                                                    \
  if (gelu) QSA_GLU(T, V, QSA_ACT_GELU); else QSA_GLU(T, V, QSA_ACT_SILU)
  if (f32) { if (vec) { QSA_GLU_A(float, 8); } else { QSA_GLU_A(float, 1); } }
  else     { if (vec) { QSA_GLU_A(bf16_t, 8); } else { QSA_GLU_A(bf16_t, 1); } }
#undef QSA_GLU_A
#undef QSA_GLU
}

// ---------------------------------------------------------------------------
// Latent norms of one projected row, both RMS with a plain weight:
//   blockIdx.y == 0: cq[row]        = rms(x[row, :qr]) * wq
//   blockIdx.y == 1: cache[slot]    = rms(x[row, qr:qr+kr]) * wk
// slot = page*64 + offset of the row's position; negative slots are skipped.
// ---------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256)
qsa_latent_norm_store(const T* __restrict__ x, long long xstride,
                      const T* __restrict__ wq, const T* __restrict__ wk,
                      T* __restrict__ cq, T* __restrict__ cache,
                      const int* __restrict__ slots, int qr, int kr,
                      float eps) {
  __shared__ float scratch[8];
  const long long row = blockIdx.x;
  const bool lat = blockIdx.y == 1;
  const int n = lat ? kr : qr;
  const T* src = x + row * xstride + (lat ? qr : 0);
  const T* w = lat ? wk : wq;
  T* dst = cq + row * qr;
  if (lat) {
    const int slot = slots[row];
    if (slot < 0) return;                       // uniform over the block
    dst = cache + (long long)slot * kr;
  }
  float ss = 0.f;
  for (int i = threadIdx.x; i < n; i += blockDim.x) {
    const float v = ldf<T>(src + i);
    ss = fmaf(v, v, ss);
  }
  ss = block_reduce_sum(ss, scratch);
  const float inv = 1.f / sqrtf(ss / (float)n + eps);
  for (int i = threadIdx.x; i < n; i += blockDim.x)
    stf<T>(dst + i, ldf<T>(src + i) * inv * ldf<T>(w + i));
}

extern "C" void qsa_latent_norm_store_launch(
    const void* x, long long xstride, const void* wq, const void* wk,
    void* cq, void* cache, const int* slots, long long rows, int qr, int kr,
    float eps, int f32, hipStream_t st) {
  dim3 grid((unsigned)rows, 2);
  if (f32)
    hipLaunchKernelGGL((qsa_latent_norm_store<float>), grid, dim3(256), 0, st,
                       (const float*)x, xstride, (const float*)wq,
                       (const float*)wk, (float*)cq, (float*)cache, slots, qr,
                       kr, eps);
  else
    hipLaunchKernelGGL((qsa_latent_norm_store<bf16_t>), grid, dim3(256), 0,
                       st, (const bf16_t*)x, xstride, (const bf16_t*)wq,
                       (const bf16_t*)wk, (bf16_t*)cq, (bf16_t*)cache, slots,
                       qr, kr, eps);
}

// ---------------------------------------------------------------------------
// Cache slot of every decode row's newest position (-1: row not in use).
// ---------------------------------------------------------------------------
__global__ void qsa_decode_slots(const int* __restrict__ block_table,
                                 const int* __restrict__ seq_lens,
                                 int* __restrict__ slots, int B,
                                 int max_pages) {
  const int b = blockIdx.x * blockDim.x + threadIdx.x;
  if (b >= B) return;
  const int p = seq_lens[b] - 1;
  slots[b] = (p < 0 || p / 64 >= max_pages)
                 ? -1
                 : block_table[(long long)b * max_pages + p / 64] * 64 +
                       p % 64;
}

extern "C" void qsa_decode_slots_launch(const int* block_table,
                                        const int* seq_lens, int* slots,
                                        int B, int max_pages,
                                        hipStream_t st) {
  hipLaunchKernelGGL(qsa_decode_slots, dim3((B + 63) / 64), dim3(64), 0, st,
                     block_table, seq_lens, slots, B, max_pages);
}

// ---------------------------------------------------------------------------
// Greedy pick: index of the largest logit of each row, the lowest index on
// ties.  One block per row and no scratch memory to clear, so it can be
// recorded into a graph.
// ---------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(1024)
qsa_argmax_rows(const T* __restrict__ x, long long* __restrict__ out, int n) {
  __shared__ float sv[16];
  __shared__ int si[16];
  const T* r = x + (long long)blockIdx.x * n;
  float best = -INFINITY;
  int at = 0x7fffffff;
  for (int i = threadIdx.x; i < n; i += blockDim.x) {
    const float v = ldf<T>(r + i);
    if (v > best || at == 0x7fffffff) { best = v; at = i; }
  }
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) {
    const float v = __shfl_xor(best, off, QSA_WAVE);
    const int i = __shfl_xor(at, off, QSA_WAVE);
    if (v > best || (v == best && i < at)) { best = v; at = i; }
  }
  const int wave = threadIdx.x >> 6;
  if ((threadIdx.x & 63) == 0) { sv[wave] = best; si[wave] = at; }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int k = 1; k < (int)(blockDim.x >> 6); ++k)
      if (sv[k] > best || (sv[k] == best && si[k] < at)) {
        best = sv[k];
        at = si[k];
      }
    out[blockIdx.x] = at < n ? at : 0;
  }
}

extern "C" void qsa_argmax_rows_launch(const void* x, long long* out,
                                       long long rows, int n, int f32,
                                       hipStream_t st) {
  if (f32)
    hipLaunchKernelGGL((qsa_argmax_rows<float>), dim3((unsigned)rows),
                       dim3(1024), 0, st, (const float*)x, out, n);
  else
    hipLaunchKernelGGL((qsa_argmax_rows<bf16_t>), dim3((unsigned)rows),
                       dim3(1024), 0, st, (const bf16_t*)x, out, n);
}
