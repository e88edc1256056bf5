// Latent attention (one cached latent per token shared by all heads) with an
// optional sliding window, a per-head softmax sink and an output gate.
//
// Cache: [pages, 64, KR], row-major; k = Wuk c and v = Wuv c are never
// cached.  Two ways through it, same result up to rounding:
//   absorbed  q' = Wuk^T q per head, scores q'.c, read-out sum p c, then
//             Wuv per head.  Reads only latents: decode rows and short
//             portions.            (qsa_head_matmul, qsa_latent_rows*)
//   expanded  k and v of the visible context materialized by one GEMM,
//             flash attention over them: prompt portions.
//                                   (qsa_window_attn_prefill)
// Window: position i sees j with 0 <= i - j < size.  The softmax sink adds
// exp(sink_h) to the denominator: no key, no value, no scale.
#include "lm_common.h"

#define LPAGE 64
#define NEG_BIG (-3.0e38f)
#define LOG2E 1.4426950408889634f

// ---------------------------------------------------------------------------
// Per-head product: out[m, h, n] = sum_k x[m, h, k] W[h, n, k], optionally
// times sigmoid(gate[m, h*N + n]).
// ---------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256)
qsa_head_matmul(const T* __restrict__ x, long long xrow,
                const T* __restrict__ W, const T* __restrict__ gate,
                long long grow, T* __restrict__ out, int H, int N, int K) {
  extern __shared__ float xs[];
  const long long m = blockIdx.x / H;
  const int h = blockIdx.x % H;
  const T* xr = x + m * xrow + (long long)h * K;
  for (int k = threadIdx.x; k < K; k += blockDim.x) xs[k] = ldf<T>(xr + k);
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  for (int n = wave; n < N; n += (int)(blockDim.x >> 6)) {
    const T* w = W + ((long long)h * N + n) * K;
    float a = 0.f;
    for (int k = lane; k < K; k += 64) a = fmaf(xs[k], ldf<T>(w + k), a);
    a = wave_reduce_sum(a);
    if (lane == 0) {
      if (gate) a *= sigmoid_f(ldf<T>(gate + m * grow + (long long)h * N + n));
      stf<T>(out + (m * H + h) * N + n, a);
    }
  }
}

// Matrix cores.  A wave computes 16 columns of one head for up to 64 rows; W
// rows are the A operand, so a lane ends up with 4 consecutive columns of one
// row.  SPLIT: the four waves of a block share the columns, split K (every
// load of the product is in flight at once) and meet in LDS; otherwise they
// take 16 columns each.
template <bool SPLIT>
__global__ void __launch_bounds__(256)
qsa_head_matmul_mfma(const bf16_t* __restrict__ x, long long xrow,
                     const bf16_t* __restrict__ W,
                     const bf16_t* __restrict__ gate, long long grow,
                     bf16_t* __restrict__ out, int M, int H, int N, int K,
                     int NT) {
  __shared__ f32x4_v red[SPLIT ? 4 : 1][4][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int col = lane & 15, hi = lane >> 4;
  const int nt = SPLIT ? blockIdx.x % NT : blockIdx.x % NT * 4 + wave;
  const int h = (blockIdx.x / NT) % H;
  const int m0 = (blockIdx.x / (NT * H)) * 64;
  const int nmt = min(4, (M - m0 + 15) / 16);
  const bf16_t* xr[4];
#pragma unroll
  for (int t = 0; t < 4; ++t)
    xr[t] = x + (long long)min(m0 + t * 16 + col, M - 1) * xrow +
            (long long)h * K;
  const bf16_t* wr = W + ((long long)h * N + min(nt * 16 + col, N - 1)) * K;
  const bf16x8_v zero = {0, 0, 0, 0, 0, 0, 0, 0};
  f32x4_v acc[4];
#pragma unroll
  for (int t = 0; t < 4; ++t) acc[t] = (f32x4_v){0.f, 0.f, 0.f, 0.f};
  const int per = SPLIT ? ((K + 31) / 32 + 3) / 4 * 32 : K;
  const int ka = SPLIT ? wave * per : 0;
  const int k1 = min(K, ka + per);
  for (int k0 = ka; k0 < k1; k0 += 128) {
    bf16x8_v a[4];
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const int k = k0 + s * 32 + hi * 8;           // K % 8 == 0
      const bf16x8_v v = *reinterpret_cast<const bf16x8_v*>(
          wr + (k < k1 ? k : 0));
      a[s] = k < k1 ? v : zero;
    }
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      if (t >= nmt) break;                          // uniform
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        const int k = k0 + s * 32 + hi * 8;
        bf16x8_v b = *reinterpret_cast<const bf16x8_v*>(
            xr[t] + (k < k1 ? k : 0));
        b = k < k1 ? b : zero;
        acc[t] = mfma_bf16(a[s], b, acc[t]);
      }
    }
  }
  const int n0 = nt * 16 + hi * 4;
  auto finish = [&](int m, f32x4_v s) {
    if (m >= M || n0 >= N) return;                  // N % 4 == 0
    float v[4] = {s[0], s[1], s[2], s[3]};
    if (gate) {
      float g[4];
      ldv<bf16_t, 4>(gate + (long long)m * grow + (long long)h * N + n0, g);
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] /= 1.f + __expf(-g[r]);
    }
    stv<bf16_t, 4>(out + ((long long)m * H + h) * N + n0, v);
  };
  if (SPLIT) {
#pragma unroll
    for (int t = 0; t < 4; ++t) red[wave][t][lane] = acc[t];
    lds_barrier();
    finish(m0 + wave * 16 + col,
           (red[0][wave][lane] + red[1 % (SPLIT ? 4 : 1)][wave][lane]) +
               (red[2 % (SPLIT ? 4 : 1)][wave][lane] +
                red[3 % (SPLIT ? 4 : 1)][wave][lane]));
  } else {
#pragma unroll
    for (int t = 0; t < 4; ++t) finish(m0 + t * 16 + col, acc[t]);
  }
}

extern "C" void qsa_head_matmul_launch(const void* x, long long xrow,
                                       const void* W, const void* gate,
                                       long long grow, void* out, int M,
                                       int H, int N, int K, int f32,
                                       int mfma, hipStream_t st) {
  if (mfma) {
    const bool split = K > 128;
    const int NT = split ? (N + 15) / 16 : (N + 63) / 64;
    dim3 grid((unsigned)((M + 63) / 64 * H * NT));
    auto* kernel = split ? qsa_head_matmul_mfma<true>
                         : qsa_head_matmul_mfma<false>;
    hipLaunchKernelGGL(kernel, grid, dim3(256), 0, st,
                       (const bf16_t*)x, xrow, (const bf16_t*)W,
                       (const bf16_t*)gate, grow, (bf16_t*)out, M, H, N, K,
                       NT);
    return;
  }
  dim3 grid((unsigned)((long long)M * H));
  if (f32)
    hipLaunchKernelGGL((qsa_head_matmul<float>), grid, dim3(256),
                       sizeof(float) * K, st, (const float*)x, xrow,
                       (const float*)W, (const float*)gate, grow,
                       (float*)out, H, N, K);
  else
    hipLaunchKernelGGL((qsa_head_matmul<bf16_t>), grid, dim3(256),
                       sizeof(float) * K, st, (const bf16_t*)x, xrow,
                       (const bf16_t*)W, (const bf16_t*)gate, grow,
                       (bf16_t*)out, H, N, K);
}

// ---------------------------------------------------------------------------
// Absorbed attention of single rows, any size and storage type: one block
// per (row, head).  out[row, h, KR] = softmax-with-sink(q'.c * scale) c.
// ---------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256)
qsa_latent_rows(const T* __restrict__ qa, const T* __restrict__ cache,
                const int* __restrict__ block_table, int max_pages,
                const int* __restrict__ row_item,
                const int* __restrict__ row_len, const T* __restrict__ sink,
                T* __restrict__ out, int H, int KR, int window, float scale) {
  extern __shared__ float sm[];
  float* qs = sm;              // KR
  float* os = qs + KR;         // KR
  __shared__ float sc[LPAGE];
  const long long row = blockIdx.x / H;
  const int h = blockIdx.x % H;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const T* q = qa + (row * H + h) * KR;
  T* orow = out + (row * H + h) * KR;
  for (int k = tid; k < KR; k += 256) {
    qs[k] = ldf<T>(q + k);
    os[k] = 0.f;
  }
  int n = row_len[row];
  n = n > max_pages * LPAGE ? max_pages * LPAGE : n;
  const int lo = window > 0 ? max(0, n - window) : 0;
  const int* bt = block_table +
                  (long long)(row_item ? row_item[row] : row) * max_pages;
  float m = NEG_BIG, l = 0.f;
  __syncthreads();
  for (int pg = lo / LPAGE; pg * LPAGE < n; ++pg) {
    const T* base = cache + (long long)bt[pg] * LPAGE * KR;
    const int a = max(lo - pg * LPAGE, 0), b = min(n - pg * LPAGE, LPAGE);
    for (int j = wave; j < LPAGE; j += 4) {
      float s = 0.f;
      if (j >= a && j < b) {
        for (int k = lane; k < KR; k += 64)
          s = fmaf(qs[k], ldf<T>(base + (long long)j * KR + k), s);
        s = wave_reduce_sum(s) * scale;
      } else {
        s = NEG_BIG;
      }
      if (lane == 0) sc[j] = s;
    }
    __syncthreads();
    const float mn = fmaxf(m, wave_reduce_max(sc[lane]));
    const float alpha = m > NEG_BIG ? expf(m - mn) : 0.f;
    const float p = sc[lane] > NEG_BIG ? expf(sc[lane] - mn) : 0.f;
    l = l * alpha + wave_reduce_sum(p);
    m = mn;
    for (int k = tid; k < KR; k += 256) {
      float acc = os[k] * alpha;
      for (int j = a; j < b; ++j)
        acc = fmaf(expf(sc[j] - mn), ldf<T>(base + (long long)j * KR + k),
                   acc);
      os[k] = acc;
    }
    __syncthreads();
  }
  const float sk = ldf<T>(sink + h);
  const float top = fmaxf(m, sk);
  const float f = m > NEG_BIG ? expf(m - top) : 0.f;
  const float inv = f / (l * f + expf(sk - top));
  for (int k = tid; k < KR; k += 256) stf<T>(orow + k, os[k] * inv);
}

extern "C" void qsa_latent_rows_launch(
    const void* qa, const void* cache, const int* block_table, int max_pages,
    const int* row_item, const int* row_len, const void* sink, void* out,
    int R, int H, int KR, int window, float scale, int f32, hipStream_t st) {
  dim3 grid((unsigned)((long long)R * H));
  const size_t lds = sizeof(float) * 2 * (size_t)KR;
  if (f32)
    hipLaunchKernelGGL((qsa_latent_rows<float>), grid, dim3(256), lds, st,
                       (const float*)qa, (const float*)cache, block_table,
                       max_pages, row_item, row_len, (const float*)sink,
                       (float*)out, H, KR, window, scale);
  else
    hipLaunchKernelGGL((qsa_latent_rows<bf16_t>), grid, dim3(256), lds, st,
                       (const bf16_t*)qa, (const bf16_t*)cache, block_table,
                       max_pages, row_item, row_len, (const bf16_t*)sink,
                       (bf16_t*)out, H, KR, window, scale);
}

// ---------------------------------------------------------------------------
// Absorbed attention on the matrix cores: block = (row, 16 heads, split of
// the visible pages), the page tile in LDS read once from HBM.
//   scores: wave w computes positions 16w..16w+15 x 16 heads
//           (A = latent rows, B = absorbed queries held in registers)
//   read-out: wave w owns 16*DTW latent columns; A = transposed LDS reads of
//           the same tile, B = P^T exactly as the score product left it,
//           exchanged between the waves through 2 KiB of LDS.
// Softmax statistics are shared by the block; partials (o, m, l) of the
// splits meet in qsa_latent_merge, which also adds the sink.
// ---------------------------------------------------------------------------
template <int DTW>  // latent columns <= 64 * DTW
__global__ void __launch_bounds__(256, 2)
qsa_latent_rows_mfma(const bf16_t* __restrict__ qa,
                     const bf16_t* __restrict__ cache,
                     const int* __restrict__ block_table, int max_pages,
                     const int* __restrict__ row_item,
                     const int* __restrict__ row_len,
                     float* __restrict__ part_o, float* __restrict__ part_ml,
                     int H, int KR, int window, float scale2, int NS) {
  constexpr int DP = 64 * DTW;
  constexpr int CP = DP + 16;
  constexpr int KS = DP / 32;
  constexpr int LD = LPAGE * DP / 8 / 256;
  __shared__ __attribute__((aligned(16))) bf16_t ct[LPAGE * CP];
  __shared__ __attribute__((aligned(16))) uint2 ps[4][64];
  __shared__ float smax[4][16];
  const int HT = (H + 15) / 16;
  const int split = blockIdx.x % NS;
  const int ht = (blockIdx.x / NS) % HT;
  const long long row = blockIdx.x / ((long long)NS * HT);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int col = lane & 15, hi = lane >> 4;
  const int head = ht * 16 + col;
  const int n = min(row_len[row], max_pages * LPAGE);
  const int lo = window > 0 ? max(0, n - window) : 0;
  const int pg0 = lo / LPAGE;
  const int np = n > 0 ? (n + LPAGE - 1) / LPAGE - pg0 : 0;
  const int per = (np + NS - 1) / NS;
  const int pa = pg0 + split * per;
  const int pb = min(pg0 + np, pa + per);
  const int* bt = block_table +
                  (long long)(row_item ? row_item[row] : row) * max_pages;

  float m = NEG_BIG, l = 0.f;
  f32x4_v acc[DTW];
#pragma unroll
  for (int t = 0; t < DTW; ++t) acc[t] = (f32x4_v){0.f, 0.f, 0.f, 0.f};

  if (pa < pb) {                                    // uniform over the block
    const bf16_t* qr = qa + (row * H + min(head, H - 1)) * KR;
    const bf16x8_v zero = {0, 0, 0, 0, 0, 0, 0, 0};
    bf16x8_v qf[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int k = s * 32 + hi * 8;                // KR % 8 == 0
      bf16x8_v v = *reinterpret_cast<const bf16x8_v*>(qr + (k < KR ? k : 0));
      qf[s] = k < KR ? v : zero;
    }
    uint4 reg[LD];
    auto fetch = [&](int pg) {
      const bf16_t* base = cache + (long long)bt[pg] * LPAGE * KR;
      const int a = lo - pg * LPAGE, b = n - pg * LPAGE;
#pragma unroll
      for (int u = 0; u < LD; ++u) {
        const int g = tid + u * 256;
        const int r = g / (DP / 8), c = (g % (DP / 8)) * 8;
        const bool ok = c < KR && r >= a && r < b;
        const uint4 v = *reinterpret_cast<const uint4*>(
            base + (unsigned)(ok ? r * KR + c : 0));
        reg[u] = ok ? v : make_uint4(0, 0, 0, 0);
      }
    };
    fetch(pa);
    for (int pg = pa; pg < pb; ++pg) {
      lds_barrier();                              // readers of ct/ps done
#pragma unroll
      for (int u = 0; u < LD; ++u) {
        const int g = tid + u * 256;
        const int r = g / (DP / 8), c = (g % (DP / 8)) * 8;
        *reinterpret_cast<uint4*>(&ct[r * CP + c]) = reg[u];
      }
      lds_barrier();
      if (pg + 1 < pb) fetch(pg + 1);
      f32x4_v s4 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const bf16x8_v a = *reinterpret_cast<const bf16x8_v*>(
            &ct[(wave * 16 + col) * CP + s * 32 + hi * 8]);
        s4 = mfma_bf16(a, qf[s], s4);
      }
      float mx = NEG_BIG;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int p = pg * LPAGE + wave * 16 + hi * 4 + r;
        s4[r] = (p >= lo && p < n) ? s4[r] * scale2 : NEG_BIG;
        mx = fmaxf(mx, s4[r]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, QSA_WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, QSA_WAVE));
      if (hi == 0) smax[wave][col] = mx;
      lds_barrier();
      float mn = m;
#pragma unroll
      for (int w = 0; w < 4; ++w) mn = fmaxf(mn, smax[w][col]);
      const float alpha = m > NEG_BIG ? exp2f(m - mn) : 0.f;
      m = mn;
      float p[4];
#pragma unroll
      for (int r = 0; r < 4; ++r)
        p[r] = s4[r] > NEG_BIG ? exp2f(s4[r] - mn) : 0.f;
      l = l * alpha + (p[0] + p[1]) + (p[2] + p[3]);
      ps[wave][lane] =
          make_uint2(cvt_bf16x2(p[0], p[1]), cvt_bf16x2(p[2], p[3]));
#pragma unroll
      for (int t = 0; t < DTW; ++t) acc[t] *= alpha;
      lds_barrier();
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        const uint2 x0 = ps[s * 2][lane], x1 = ps[s * 2 + 1][lane];
        const uint4 xx = make_uint4(x0.x, x0.y, x1.x, x1.y);
        const bf16x8_v pf = __builtin_bit_cast(bf16x8_v, xx);
#pragma unroll
        for (int t = 0; t < DTW; ++t) {
          const bf16x8_v a = lds_frag_tr(ct, CP, s * 32, s * 32 + 16,
                                         (wave * DTW + t) * 16, lane);
          acc[t] = mfma_bf16(a, pf, acc[t]);
        }
      }
    }
  }
  // l: sum over the hi groups of each wave, then over the waves
  l += __shfl_xor(l, 16, QSA_WAVE);
  l += __shfl_xor(l, 32, QSA_WAVE);
  lds_barrier();
  if (hi == 0) smax[wave][col] = l;
  lds_barrier();
  if (head < H) {
    const long long o = (row * H + head) * NS + split;
    if (wave == 0 && hi == 0) {
      part_ml[o * 2] = m;
      part_ml[o * 2 + 1] =
          (smax[0][col] + smax[1][col]) + (smax[2][col] + smax[3][col]);
    }
#pragma unroll
    for (int t = 0; t < DTW; ++t) {
      const int d = (wave * DTW + t) * 16 + hi * 4;
      if (d < KR)
        *reinterpret_cast<float4*>(part_o + o * KR + d) =
            make_float4(acc[t][0], acc[t][1], acc[t][2], acc[t][3]);
    }
  }
}

// Splits -> normalized read-out; the sink joins the denominator here.
// m and the sink are in powers of two.
__global__ void __launch_bounds__(256)
qsa_latent_merge(const float* __restrict__ part_o,
                 const float* __restrict__ part_ml,
                 const bf16_t* __restrict__ sink, bf16_t* __restrict__ out,
                 int H, int KR, int NS) {
  extern __shared__ float ws[];                     // NS weights
  const long long rh = blockIdx.x;
  const float* ml = part_ml + rh * NS * 2;
  const float sk = bf16_to_f32(sink[rh % H]) * LOG2E;
  const int lane = threadIdx.x & 63;
  float top = NEG_BIG;
  for (int s = lane; s < NS; s += 64)
    if (ml[2 * s + 1] > 0.f) top = fmaxf(top, ml[2 * s]);
  top = fmaxf(wave_reduce_max(top), sk);
  float den = 0.f;
  for (int s = lane; s < NS; s += 64) {
    const float w = ml[2 * s + 1] > 0.f ? exp2f(ml[2 * s] - top) : 0.f;
    if (threadIdx.x < 64) ws[s] = w;
    den = fmaf(w, ml[2 * s + 1], den);
  }
  const float inv = 1.f / (wave_reduce_sum(den) + exp2f(sk - top));
  __syncthreads();
  for (int k = threadIdx.x * 4; k < KR; k += blockDim.x * 4) {
    f32x4_v a = {0.f, 0.f, 0.f, 0.f};
    const float* po = part_o + rh * NS * KR + k;
#pragma unroll 8
    for (int s = 0; s < NS; ++s)
      a += ws[s] * *reinterpret_cast<const f32x4_v*>(po + (long long)s * KR);
    float v[4] = {a[0] * inv, a[1] * inv, a[2] * inv, a[3] * inv};
    stv<bf16_t, 4>(out + rh * KR + k, v);
  }
}

extern "C" void qsa_latent_rows_mfma_launch(
    const bf16_t* qa, const bf16_t* cache, const int* block_table,
    int max_pages, const int* row_item, const int* row_len,
    const bf16_t* sink, float* part_o, float* part_ml, bf16_t* out, int R,
    int H, int KR, int window, float scale, int NS, hipStream_t st) {
  dim3 grid((unsigned)((long long)R * ((H + 15) / 16) * NS));
  const float scale2 = scale * LOG2E;
#define QSA_LR(D)                                                           \
  hipLaunchKernelGGL((qsa_latent_rows_mfma<D>), grid, dim3(256), 0, st, qa, \
                     cache, block_table, max_pages, row_item, row_len,      \
                     part_o, part_ml, H, KR, window, scale2, NS)
  if (KR <= 64) QSA_LR(1);
  else if (KR <= 128) QSA_LR(2);
  else if (KR <= 256) QSA_LR(4);
  else QSA_LR(8);
#undef QSA_LR
  const int th = KR >= 1024 ? 256 : (KR / 4 + 63) / 64 * 64;
  hipLaunchKernelGGL(qsa_latent_merge, dim3((unsigned)((long long)R * H)),
                     dim3(th), sizeof(float) * NS, st, part_o, part_ml, sink,
                     out, H, KR, NS);
}

// ---------------------------------------------------------------------------
// Windowed flash attention of prompt portions over expanded keys/values.
// Block = (64-row query block, head): wave w owns 16 rows; 64-key tiles of K
// and V go through LDS once per block.  O^T stays in accumulators (row =
// value column, column = query row), so the softmax state, the rescale and
// P^T (B operand of the second product) are all lane-local.
//   q   [rows, H, D]           row stride qstride
//   kv  [context rows, H*(D+E)]: k of head h at h*D, v at H*D + h*E
//   portion it: rows off..off+len-1 at positions start..; its context rows
//   begin at ctx_off and hold positions ctx_pos..start+len-1.
// ---------------------------------------------------------------------------
template <int KS, int ET>  // D <= 32*KS, E <= 16*ET
__global__ void __launch_bounds__(256, ET <= 8 ? 2 : 1)
qsa_window_attn_prefill(const bf16_t* __restrict__ q, long long qstride,
                        const bf16_t* __restrict__ kv, long long kvstride,
                        const bf16_t* __restrict__ gate, long long gstride,
                        const bf16_t* __restrict__ sink,
                        const int* __restrict__ qb_item,
                        const int* __restrict__ qb_t0,
                        const int* __restrict__ off,
                        const int* __restrict__ start,
                        const int* __restrict__ len,
                        const int* __restrict__ ctx_off,
                        const int* __restrict__ ctx_pos,
                        bf16_t* __restrict__ out, int H, int D, int E,
                        int window, float scale2) {
  constexpr int KP = 32 * KS + 8;
  constexpr int VP = 16 * ET + 16;
  constexpr int KG = 4 * KS, VG = 2 * ET;         // 16 B groups per row
  constexpr int KL = 64 * KG / 256, VL = (64 * VG + 255) / 256;
  __shared__ __attribute__((aligned(16))) bf16_t kt[64 * KP];
  __shared__ __attribute__((aligned(16))) bf16_t vt[64 * VP];
  const int h = blockIdx.x % H;
  const int qb = blockIdx.x / H;
  const int it = qb_item[qb], t0 = qb_t0[qb];
  const int n = len[it], p0 = start[it], r0 = off[it];
  const int c_pos = ctx_pos[it];
  const long long c_off = ctx_off[it];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int col = lane & 15, hi = lane >> 4;
  const int i = t0 + wave * 16 + col;             // row within the portion
  const int qpos = p0 + i;
  const long long qrow = r0 + min(i, n - 1);

  const bf16x8_v zero = {0, 0, 0, 0, 0, 0, 0, 0};
  bf16x8_v qf[KS];
#pragma unroll
  for (int s = 0; s < KS; ++s) {
    const int d = s * 32 + hi * 8;                // D % 8 == 0
    bf16x8_v v = *reinterpret_cast<const bf16x8_v*>(
        q + qrow * qstride + (long long)h * D + (d < D ? d : 0));
    qf[s] = d < D ? v : zero;
  }
  f32x4_v acc[ET];
#pragma unroll
  for (int t = 0; t < ET; ++t) acc[t] = (f32x4_v){0.f, 0.f, 0.f, 0.f};
  float m = NEG_BIG, l = 0.f;

  // visible context rows of the block, and of this wave
  const int last = p0 + min(t0 + 63, n - 1);
  const int first = window > 0 ? max(c_pos, p0 + t0 - window + 1) : c_pos;
  const int wfirst = window > 0 ? p0 + t0 + wave * 16 - window + 1 : c_pos;
  const int wlast = p0 + t0 + wave * 16 + 15;
  const long long koff = c_off - c_pos;           // + position = kv row

  uint4 kr[KL], vr[VL];
  auto fetch = [&](int pos) {
#pragma unroll
    for (int u = 0; u < KL; ++u) {
      const int g = tid + u * 256;
      const int r = g / KG, c = (g % KG) * 8;
      const bool ok = pos + r <= last && c < D;
      const uint4 v = *reinterpret_cast<const uint4*>(
          kv + (koff + min(pos + r, last)) * kvstride + (long long)h * D +
          (c < D ? c : 0));
      kr[u] = ok ? v : make_uint4(0, 0, 0, 0);
    }
#pragma unroll
    for (int u = 0; u < VL; ++u) {
      const int g = tid + u * 256;
      const int r = g / VG, c = (g % VG) * 8;
      const bool ok = pos + r <= last && c < E;
      const uint4 v = *reinterpret_cast<const uint4*>(
          kv + (koff + min(pos + r, last)) * kvstride + (long long)H * D +
          (long long)h * E + (c < E ? c : 0));
      vr[u] = ok ? v : make_uint4(0, 0, 0, 0);
    }
  };
  fetch(first);
  for (int pos = first; pos <= last; pos += 64) {
    lds_barrier();
#pragma unroll
    for (int u = 0; u < KL; ++u) {
      const int g = tid + u * 256;
      *reinterpret_cast<uint4*>(&kt[(g / KG) * KP + (g % KG) * 8]) = kr[u];
    }
#pragma unroll
    for (int u = 0; u < VL; ++u) {
      const int g = tid + u * 256;
      if (g < 64 * VG)
        *reinterpret_cast<uint4*>(&vt[(g / VG) * VP + (g % VG) * 8]) = vr[u];
    }
    lds_barrier();
    if (pos + 64 <= last) fetch(pos + 64);
    if (pos > wlast || pos + 63 < wfirst) continue;   // nothing for this wave
    f32x4_v s4[4];
    float mx = NEG_BIG;
#pragma unroll
    for (int pt = 0; pt < 4; ++pt) {
      f32x4_v a4 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const bf16x8_v a = *reinterpret_cast<const bf16x8_v*>(
            &kt[(pt * 16 + col) * KP + s * 32 + hi * 8]);
        a4 = mfma_bf16(a, qf[s], a4);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int p = pos + pt * 16 + hi * 4 + r;
        const bool ok = p <= qpos && p <= last &&
                        (window <= 0 || qpos - p < window);
        a4[r] = ok ? a4[r] * scale2 : NEG_BIG;
        mx = fmaxf(mx, a4[r]);
      }
      s4[pt] = a4;
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, QSA_WAVE));
    mx = fmaxf(mx, __shfl_xor(mx, 32, QSA_WAVE));
    const float mn = fmaxf(m, mx);
    const float alpha = m > NEG_BIG ? exp2f(m - mn) : 0.f;
    m = mn;
    float psum = 0.f;
    bf16x8_v pf[2];
#pragma unroll
    for (int pt = 0; pt < 4; ++pt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float p = s4[pt][r] > NEG_BIG ? exp2f(s4[pt][r] - mn) : 0.f;
        psum += p;
        pf[pt >> 1][(pt & 1) * 4 + r] = (short)cvt_bf16(p);
      }
    l = l * alpha + psum;
#pragma unroll
    for (int t = 0; t < ET; ++t) acc[t] *= alpha;
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int t = 0; t < ET; ++t) {
        const bf16x8_v a =
            lds_frag_tr(vt, VP, s * 32, s * 32 + 16, t * 16, lane);
        acc[t] = mfma_bf16(a, pf[s], acc[t]);
      }
  }
  l += __shfl_xor(l, 16, QSA_WAVE);
  l += __shfl_xor(l, 32, QSA_WAVE);
  const float sk = bf16_to_f32(sink[h]) * LOG2E;
  const float top = fmaxf(m, sk);
  const float f = m > NEG_BIG ? exp2f(m - top) : 0.f;
  const float inv = f / (l * f + exp2f(sk - top));
  if (i < n) {
    const bf16_t* g = gate + (long long)(r0 + i) * gstride + (long long)h * E;
    bf16_t* orow = out + ((long long)(r0 + i) * H + h) * E;
#pragma unroll
    for (int t = 0; t < ET; ++t) {
      const int e = t * 16 + hi * 4;
      if (e < E) {                                  // E % 8 == 0
        float gv[4], o[4];
        ldv<bf16_t, 4>(g + e, gv);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          o[r] = acc[t][r] * inv / (1.f + __expf(-gv[r]));
        stv<bf16_t, 4>(orow + e, o);
      }
    }
  }
}

extern "C" void qsa_window_attn_prefill_launch(
    const bf16_t* q, long long qstride, const bf16_t* kv, long long kvstride,
    const bf16_t* gate, long long gstride, const bf16_t* sink,
    const int* qb_item, const int* qb_t0, const int* off, const int* start,
    const int* len, const int* ctx_off, const int* ctx_pos, bf16_t* out,
    int QB, int H, int D, int E, int window, float scale, hipStream_t st) {
  dim3 grid((unsigned)((long long)QB * H));
  const float scale2 = scale * LOG2E;
#define QSA_WA(K, V)                                                         \
  hipLaunchKernelGGL((qsa_window_attn_prefill<K, V>), grid, dim3(256), 0,    \
                     st, q, qstride, kv, kvstride, gate, gstride, sink,      \
                     qb_item, qb_t0, off, start, len, ctx_off, ctx_pos, out, \
                     H, D, E, window, scale2)
#define QSA_WA_E(K)                                                          \
  if (E <= 32) QSA_WA(K, 2);                                                 \
  else if (E <= 64) QSA_WA(K, 4);                                            \
  else if (E <= 128) QSA_WA(K, 8);                                           \
  else QSA_WA(K, 16)
  if (D <= 32) { QSA_WA_E(1); }
  else if (D <= 64) { QSA_WA_E(2); }
  else if (D <= 128) { QSA_WA_E(4); }
  else { QSA_WA_E(8); }
#undef QSA_WA_E
#undef QSA_WA
}
