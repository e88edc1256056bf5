// Grouped-query attention over paged keys and values, with a per-head softmax
// sink and an output gate; key and value sizes are independent.
//
// Pages are row-major per key head: k [pages, G, 64, D], v [pages, G, 64, E],
// so a page of a key head is one contiguous tile for both sides, and a new
// token writes whole rows.  H / G query heads read the same tile.
//   out = softmax-with-sink(q.k * scale) v * sigmoid(gate) * out_scale
// The sink adds exp(sink_h) to the denominator: no key, no value, no scale.
//
//   qsa_gqa_rows        one block per (row, head), any size and storage type
//   qsa_gqa_rows_mfma   single rows and short portions: a wave takes a share
//                       of a row's pages for up to 16 heads of a key head
//                       (+ qsa_gqa_merge)
//   qsa_gqa_portions    flash attention of longer portions, page by page
#include "lm_common.h"

#define PG 64
#define NEG_BIG (-3.0e38f)
#define LOG2E 1.4426950408889634f

// 2^x by the hardware instruction; what would be denormal becomes zero
__device__ __forceinline__ float exp2_hw(float x) {
  return __builtin_amdgcn_exp2f(x);
}

template <typename T>
__global__ void __launch_bounds__(256)
qsa_gqa_rows(const T* __restrict__ q, const T* __restrict__ kc,
             const T* __restrict__ vc, const int* __restrict__ block_table,
             int max_pages, const int* __restrict__ row_item,
             const int* __restrict__ row_len, const float* __restrict__ sink,
             const T* __restrict__ gate, long long gstride,
             T* __restrict__ out, long long ostride, int H, int G, int D,
             int E, float scale, float out_scale) {
  extern __shared__ float sm[];
  float* qs = sm;              // D
  float* os = qs + D;          // E
  __shared__ float sc[PG], ps[PG];
  const long long row = blockIdx.x / H;
  const int h = blockIdx.x % H, g = h / (H / G);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  for (int k = tid; k < D; k += 256) qs[k] = ldf<T>(q + (row * H + h) * D + k);
  for (int k = tid; k < E; k += 256) os[k] = 0.f;
  int n = row_len[row];
  n = n > max_pages * PG ? max_pages * PG : n;
  const int* bt = block_table +
                  (long long)(row_item ? row_item[row] : row) * max_pages;
  float m = NEG_BIG, l = 0.f;
  __syncthreads();
  for (int pg = 0; pg * PG < n; ++pg) {
    const long long tile = ((long long)bt[pg] * G + g) * PG;
    const int b = min(n - pg * PG, PG);
    for (int j = wave; j < PG; j += 4) {
      float s = NEG_BIG;
      if (j < b) {
        s = 0.f;
        for (int k = lane; k < D; k += 64)
          s = fmaf(qs[k], ldf<T>(kc + (tile + j) * D + k), s);
        s = wave_reduce_sum(s) * scale;
      }
      if (lane == 0) sc[j] = s;
    }
    __syncthreads();
    const float mn = fmaxf(m, wave_reduce_max(sc[lane]));
    const float alpha = m > NEG_BIG ? expf(m - mn) : 0.f;
    const float p = sc[lane] > NEG_BIG ? expf(sc[lane] - mn) : 0.f;
    l = l * alpha + wave_reduce_sum(p);
    m = mn;
    if (wave == 0) ps[lane] = p;
    __syncthreads();
    for (int k = tid; k < E; k += 256) {
      float acc = os[k] * alpha;
      for (int j = 0; j < b; ++j)
        acc = fmaf(ps[j], ldf<T>(vc + (tile + j) * E + k), acc);
      os[k] = acc;
    }
  }
  const float sk = sink ? sink[h] : NEG_BIG;
  const float top = fmaxf(m, sk);
  const float f = m > NEG_BIG ? expf(m - top) : 0.f;
  const float den = l * f + (sink ? expf(sk - top) : 0.f);
  const float inv = den > 0.f ? f / den * out_scale : 0.f;
  for (int k = tid; k < E; k += 256) {
    float v = os[k] * inv;
    if (gate) v *= sigmoid_f(ldf<T>(gate + row * gstride + (long long)h * E + k));
    stf<T>(out + row * ostride + (long long)h * E + k, v);
  }
}

extern "C" void qsa_gqa_rows_launch(
    const void* q, const void* kc, const void* vc, const int* block_table,
    int max_pages, const int* row_item, const int* row_len, const float* sink,
    const void* gate, long long gstride, void* out, long long ostride, int R,
    int H, int G, int D, int E, float scale, float out_scale, int f32,
    hipStream_t st) {
  dim3 grid((unsigned)((long long)R * H));
  const size_t lds = sizeof(float) * ((size_t)D + E);
#define QSA_GR(T)                                                            \
  hipLaunchKernelGGL((qsa_gqa_rows<T>), grid, dim3(256), lds, st,            \
                     (const T*)q, (const T*)kc, (const T*)vc, block_table,   \
                     max_pages, row_item, row_len, sink, (const T*)gate,     \
                     gstride, (T*)out, ostride, H, G, D, E, scale, out_scale)
  if (f32) QSA_GR(float); else QSA_GR(bf16_t);
#undef QSA_GR
}

// ---------------------------------------------------------------------------
// Rows on the matrix cores.  Unit = (row, key head, 16 of its query heads,
// split of the pages), one WAVE each, no barriers: scores (A = keys straight
// from the page, B = queries in registers) leave softmax state and P^T
// lane-local (column = query head), V passes through the wave's own LDS tile
// for the transposing read.  A wave goes 32 positions at a time; the next
// keys are fetched once the scores are done, the next values once these are
// in LDS.
// ---------------------------------------------------------------------------
template <int KS, int ET>  // D <= 32*KS, E <= 16*ET
__global__ void __launch_bounds__(256, KS <= 4 && ET <= 8 ? 2 : 1)
qsa_gqa_rows_mfma(const bf16_t* __restrict__ q, const bf16_t* __restrict__ kc,
                  const bf16_t* __restrict__ vc,
                  const int* __restrict__ block_table, int max_pages,
                  const int* __restrict__ row_item,
                  const int* __restrict__ row_len,
                  float* __restrict__ part_o, float* __restrict__ part_ml,
                  int H, int G, int D, int E, float scale2, int NS,
                  int units) {
  constexpr int VP = 16 * ET + 16;
  constexpr int VG = 2 * ET;                      // 16 B groups per V row
  __shared__ __attribute__((aligned(16))) bf16_t vt_all[4][32 * VP];
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int unit = blockIdx.x * 4 + wave;
  if (unit >= units) return;
  bf16_t* vt = vt_all[wave];
  const int RG = H / G, HT = (RG + 15) / 16;
  const int split = unit % NS;
  const int ht = unit / NS % HT;
  const int g = unit / (NS * HT) % G;
  const long long row = unit / (NS * HT * G);
  const int lane = threadIdx.x & 63;
  const int col = lane & 15, hi = lane >> 4;
  const int hg = ht * 16 + col;                   // head within the group
  const int head = g * RG + min(hg, RG - 1);
  const int n = min(row_len[row], max_pages * PG);
  const int np = n > 0 ? (n + PG - 1) / PG : 0;
  const int per = (np + NS - 1) / NS;
  const int ia = split * per * 2;                 // in steps of 32 positions
  const int ib = min((n + 31) / 32, ia + per * 2);
  const int* bt = block_table +
                  (long long)(row_item ? row_item[row] : row) * max_pages;
  float m = NEG_BIG, l = 0.f;
  f32x4_v acc[ET];
#pragma unroll
  for (int t = 0; t < ET; ++t) acc[t] = (f32x4_v){0.f, 0.f, 0.f, 0.f};
  if (n > 0 && ia < ib) {                         // uniform over the wave
    const bf16x8_v zero = {0, 0, 0, 0, 0, 0, 0, 0};
    bf16x8_v qf[KS], kf[2][KS];
    u32x4_v vr[ET];
    const bf16_t* qr = q + (row * H + head) * D;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int d = s * 32 + hi * 8;              // D % 8 == 0
      const bf16x8_v v = *reinterpret_cast<const bf16x8_v*>(
          qr + (d < D ? d : 0));
      qf[s] = d < D ? v : zero;
    }
    auto fetch_k = [&](int i) {
      const bf16_t* kb = kc + (((long long)bt[i >> 1] * G + g) * PG +
                               (i & 1) * 32) * D;
#pragma unroll
      for (int pt = 0; pt < 2; ++pt)
#pragma unroll
        for (int s = 0; s < KS; ++s) {
          const int d = s * 32 + hi * 8;          // past D: times zero
          kf[pt][s] = *reinterpret_cast<const bf16x8_v*>(
              kb + (unsigned)((pt * 16 + col) * D + (d < D ? d : 0)));
        }
    };
    auto fetch_v = [&](int i) {
      const bf16_t* vb = vc + (((long long)bt[i >> 1] * G + g) * PG +
                               (i & 1) * 32) * E;
#pragma unroll
      for (int u = 0; u < ET; ++u) {
        const int k = lane + u * 64;
        const int r = k / VG, c = (k % VG) * 8;
        const bool ok = c < E && i * 32 + r < n;
        const u32x4_v v = *reinterpret_cast<const u32x4_v*>(
            vb + (unsigned)(ok ? r * E + c : 0));
        vr[u] = ok ? v : (u32x4_v){0, 0, 0, 0};
      }
    };
    fetch_k(ia);
    fetch_v(ia);
    for (int i = ia; i < ib; ++i) {
      f32x4_v s4[2];
#pragma unroll
      for (int pt = 0; pt < 2; ++pt) {
        f32x4_v a4 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KS; ++s) {
          bf16x8_v a = kf[pt][s];
          if (s * 32 + hi * 8 >= D) a = zero;
          a4 = mfma_bf16(a, qf[s], a4);
        }
        s4[pt] = a4;
      }
      if (i + 1 < ib) fetch_k(i + 1);
      __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront", "local");
      __builtin_amdgcn_wave_barrier();
#pragma unroll
      for (int u = 0; u < ET; ++u) {
        const int k = lane + u * 64;
        *reinterpret_cast<u32x4_v*>(&vt[(k / VG) * VP + (k % VG) * 8]) = vr[u];
      }
      __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront", "local");
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront", "local");
      if (i + 1 < ib) fetch_v(i + 1);
      float mx = NEG_BIG;
#pragma unroll
      for (int pt = 0; pt < 2; ++pt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int p = i * 32 + pt * 16 + hi * 4 + r;
          s4[pt][r] = p < n ? s4[pt][r] * scale2 : NEG_BIG;
          mx = fmaxf(mx, s4[pt][r]);
        }
      mx = fmaxf(mx, __shfl_xor(mx, 16, QSA_WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, QSA_WAVE));
      const float mn = fmaxf(m, mx);
      const float alpha = exp2_hw(m - mn);        // a step sees a key: mn is
                                                  // finite, masked terms 0
      m = mn;
      float psum = 0.f;
      uint2 pk[2];
#pragma unroll
      for (int pt = 0; pt < 2; ++pt) {
        float p[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          p[r] = exp2_hw(s4[pt][r] - mn);
          psum += p[r];
        }
        pk[pt] = make_uint2(cvt_bf16x2(p[0], p[1]), cvt_bf16x2(p[2], p[3]));
      }
      l = l * alpha + psum;
#pragma unroll
      for (int t = 0; t < ET; ++t) acc[t] *= alpha;
      const bf16x8_v pf = __builtin_bit_cast(
          bf16x8_v, make_uint4(pk[0].x, pk[0].y, pk[1].x, pk[1].y));
#pragma unroll
      for (int t = 0; t < ET; ++t)
        acc[t] = mfma_bf16(lds_frag_tr(vt, VP, 0, 16, t * 16, lane), pf,
                           acc[t]);
    }
    l += __shfl_xor(l, 16, QSA_WAVE);
    l += __shfl_xor(l, 32, QSA_WAVE);
  }
  if (hg < RG) {
    const long long o = (row * H + head) * NS + split;
    if (hi == 0) {
      part_ml[o * 2] = m;
      part_ml[o * 2 + 1] = l;
    }
#pragma unroll
    for (int t = 0; t < ET; ++t) {
      const int e = t * 16 + hi * 4;
      if (e < E)                                  // E % 8 == 0
        *reinterpret_cast<f32x4_v*>(part_o + o * E + e) = acc[t];
    }
  }
}

// Splits -> normalized, gated output; the sink joins the denominator here.
// Statistics are in powers of two.  WPR waves merge one (row, head): one where
// there are few splits, four that share them otherwise.
template <int WPR>
__global__ void __launch_bounds__(256)
qsa_gqa_merge(const float* __restrict__ part_o,
              const float* __restrict__ part_ml,
              const float* __restrict__ sink, const bf16_t* __restrict__ gate,
              long long gstride, bf16_t* __restrict__ out, long long ostride,
              long long total, int H, int E, int NS, float out_scale) {
  __shared__ float2 red[WPR == 1 ? 1 : WPR][64];
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int sub = wave % WPR;
  const long long rh = (long long)blockIdx.x * (4 / WPR) + wave / WPR;
  if (rh >= total) return;                        // WPR 4: never
  const int h = (int)(rh % H), lane = threadIdx.x & 63;
  const long long row = rh / H;
  const float2* ml = reinterpret_cast<const float2*>(part_ml) + rh * NS;
  const float sk = sink ? sink[h] * LOG2E : NEG_BIG;
  float top = NEG_BIG;
  for (int s = lane; s < NS; s += 64)
    if (ml[s].y > 0.f) top = fmaxf(top, ml[s].x);
  top = fmaxf(wave_reduce_max(top), sk);
  float den = 0.f;
  for (int s = lane; s < NS; s += 64)
    if (ml[s].y > 0.f) den = fmaf(exp2_hw(ml[s].x - top), ml[s].y, den);
  den = wave_reduce_sum(den) + (sink ? exp2_hw(sk - top) : 0.f);
  const float inv = den > 0.f ? out_scale / den : 0.f;
  for (int e0 = 0; e0 < E; e0 += 128) {           // E % 8 == 0
    const int e = e0 + lane * 2;
    const bool in = e < E;
    const float* po = part_o + rh * NS * E + (in ? e : 0);
    float a0 = 0.f, a1 = 0.f;
    for (int s0 = 0; s0 < NS; s0 += 64) {
      const int n = min(64, NS - s0);
      float w = 0.f;
      if (lane < n && ml[s0 + lane].y > 0.f)
        w = exp2_hw(ml[s0 + lane].x - top);
#pragma unroll 8
      for (int s = sub; s < n; s += WPR) {
        const float ws = __shfl(w, s, QSA_WAVE);
        const float2 v = *reinterpret_cast<const float2*>(
            po + (long long)(s0 + s) * E);
        a0 = fmaf(ws, v.x, a0);
        a1 = fmaf(ws, v.y, a1);
      }
    }
    if (WPR > 1) {
      red[sub % WPR][lane] = make_float2(a0, a1);
      __syncthreads();
      if (sub == 0) {
#pragma unroll
        for (int k = 1; k < WPR; ++k) {
          a0 += red[k][lane].x;
          a1 += red[k][lane].y;
        }
      }
      __syncthreads();
    }
    if (sub == 0 && in) {
      a0 *= inv;
      a1 *= inv;
      if (gate) {
        const float2 gv = bf16x2_to_f32x2(
            *reinterpret_cast<const unsigned int*>(
                gate + row * gstride + (long long)h * E + e));
        a0 /= 1.f + __expf(-gv.x);
        a1 /= 1.f + __expf(-gv.y);
      }
      *reinterpret_cast<unsigned int*>(out + row * ostride + (long long)h * E +
                                       e) = cvt_bf16x2(a0, a1);
    }
  }
}

extern "C" void qsa_gqa_rows_mfma_launch(
    const bf16_t* q, const bf16_t* kc, const bf16_t* vc,
    const int* block_table, int max_pages, const int* row_item,
    const int* row_len, const float* sink, const bf16_t* gate,
    long long gstride, float* part_o, float* part_ml, bf16_t* out,
    long long ostride, int R, int H, int G, int D, int E, float scale,
    float out_scale, int NS, hipStream_t st) {
  const int units = R * G * ((H / G + 15) / 16) * NS;
  dim3 grid((unsigned)((units + 3) / 4));
  const float scale2 = scale * LOG2E;
#define QSA_GM(K, V)                                                          \
  hipLaunchKernelGGL((qsa_gqa_rows_mfma<K, V>), grid, dim3(256), 0, st, q,    \
                     kc, vc, block_table, max_pages, row_item, row_len,       \
                     part_o, part_ml, H, G, D, E, scale2, NS, units)
#define QSA_GM_E(K)                                                           \
  if (E <= 32) QSA_GM(K, 2);                                                  \
  else if (E <= 64) QSA_GM(K, 4);                                             \
  else if (E <= 128) QSA_GM(K, 8);                                            \
  else QSA_GM(K, 16)
  if (D <= 32) { QSA_GM_E(1); }
  else if (D <= 64) { QSA_GM_E(2); }
  else if (D <= 128) { QSA_GM_E(4); }
  else { QSA_GM_E(8); }
#undef QSA_GM_E
#undef QSA_GM
  const long long total = (long long)R * H;
  if (NS > 8)
    hipLaunchKernelGGL((qsa_gqa_merge<4>), dim3((unsigned)total), dim3(256),
                       0, st, part_o, part_ml, sink, gate, gstride, out,
                       ostride, total, H, E, NS, out_scale);
  else
    hipLaunchKernelGGL((qsa_gqa_merge<1>), dim3((unsigned)((total + 3) / 4)),
                       dim3(256), 0, st, part_o, part_ml, sink, gate, gstride,
                       out, ostride, total, H, E, NS, out_scale);
}

// ---------------------------------------------------------------------------
// Flash attention of portions.  Block = (64*QT query rows, head): wave w owns
// QT tiles of 16 rows, every page tile of K and V goes through LDS once per
// block and is read by all waves, each fragment used for QT tiles.  O^T stays
// in accumulators (row = value column, column = query row), so softmax state,
// rescale and P^T are lane-local.  Blocks walk the key heads first: with G a
// multiple of the 8 dies, one die's cache keeps one key head.
// ---------------------------------------------------------------------------
template <int KS, int ET, int QT>  // D <= 32*KS, E <= 16*ET
__global__ void __launch_bounds__(256, KS <= 4 && ET <= 8 ? 2 : 1)
qsa_gqa_portions(const bf16_t* __restrict__ q, const bf16_t* __restrict__ kc,
                 const bf16_t* __restrict__ vc,
                 const int* __restrict__ block_table, int max_pages,
                 const float* __restrict__ sink,
                 const bf16_t* __restrict__ gate, long long gstride,
                 const int* __restrict__ qb_item,
                 const int* __restrict__ qb_t0, const int* __restrict__ off,
                 const int* __restrict__ start, const int* __restrict__ len,
                 bf16_t* __restrict__ out, long long ostride, int H, int G,
                 int D, int E, float scale2, float out_scale) {
  constexpr int KP = 32 * KS + 8;
  constexpr int VP = 16 * ET + 16;
  constexpr int KG = 4 * KS, VG = 2 * ET;         // 16 B groups per row
  constexpr int KL = 64 * KG / 256, VL = (64 * VG + 255) / 256;
  __shared__ __attribute__((aligned(16))) bf16_t kt[64 * KP];
  __shared__ __attribute__((aligned(16))) bf16_t vt[64 * VP];
  const int RG = H / G;
  const int g = blockIdx.x % G;
  const int h = g * RG + blockIdx.x / G % RG;
  const int qb = blockIdx.x / H;
  const int it = qb_item[qb], t0 = qb_t0[qb];
  const int n = len[it], p0 = start[it], r0 = off[it];
  const int* bt = block_table + (long long)it * max_pages;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int col = lane & 15, hi = lane >> 4;
  const int w0 = t0 + wave * 16 * QT;             // first row of this wave

  const bf16x8_v zero = {0, 0, 0, 0, 0, 0, 0, 0};
  bf16x8_v qf[QT][KS];
#pragma unroll
  for (int u = 0; u < QT; ++u) {
    const long long qrow = r0 + min(w0 + u * 16 + col, n - 1);
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int d = s * 32 + hi * 8;              // D % 8 == 0
      const bf16x8_v v = *reinterpret_cast<const bf16x8_v*>(
          q + (qrow * H + h) * D + (d < D ? d : 0));
      qf[u][s] = d < D ? v : zero;
    }
  }
  f32x4_v acc[QT][ET];
  float m[QT], l[QT];
#pragma unroll
  for (int u = 0; u < QT; ++u) {
    m[u] = NEG_BIG;
    l[u] = 0.f;
#pragma unroll
    for (int t = 0; t < ET; ++t) acc[u][t] = (f32x4_v){0.f, 0.f, 0.f, 0.f};
  }
  const int last = p0 + min(t0 + 64 * QT, n) - 1; // last visible position
  const int wlast = p0 + w0 + 16 * QT - 1;        // ... of this wave

  uint4 kr[KL], vr[VL];
  auto fetch = [&](int pg) {
    const long long tile = ((long long)bt[pg] * G + g) * PG;
    const int have = last - pg * PG;              // rows 0..have are visible
#pragma unroll
    for (int u = 0; u < KL; ++u) {
      const int i = tid + u * 256;
      const int r = i / KG, c = (i % KG) * 8;
      const bool ok = r <= have && c < D;
      const uint4 v = *reinterpret_cast<const uint4*>(
          kc + (tile + (ok ? r : 0)) * D + (ok ? c : 0));
      kr[u] = ok ? v : make_uint4(0, 0, 0, 0);
    }
#pragma unroll
    for (int u = 0; u < VL; ++u) {
      const int i = tid + u * 256;
      const int r = i / VG, c = (i % VG) * 8;
      const bool ok = r <= have && r < PG && c < E;
      const uint4 v = *reinterpret_cast<const uint4*>(
          vc + (tile + (ok ? r : 0)) * E + (ok ? c : 0));
      vr[u] = ok ? v : make_uint4(0, 0, 0, 0);
    }
  };
  fetch(0);
  for (int pg = 0; pg * PG <= last; ++pg) {
    lds_barrier();
#pragma unroll
    for (int u = 0; u < KL; ++u) {
      const int i = tid + u * 256;
      *reinterpret_cast<uint4*>(&kt[(i / KG) * KP + (i % KG) * 8]) = kr[u];
    }
#pragma unroll
    for (int u = 0; u < VL; ++u) {
      const int i = tid + u * 256;
      if (i < 64 * VG)
        *reinterpret_cast<uint4*>(&vt[(i / VG) * VP + (i % VG) * 8]) = vr[u];
    }
    lds_barrier();
    if ((pg + 1) * PG <= last) fetch(pg + 1);
    if (pg * PG > wlast) continue;                // nothing for this wave
    f32x4_v s4[QT][4];
#pragma unroll
    for (int pt = 0; pt < 4; ++pt) {
#pragma unroll
      for (int u = 0; u < QT; ++u) s4[u][pt] = (f32x4_v){0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const bf16x8_v a = *reinterpret_cast<const bf16x8_v*>(
            &kt[(pt * 16 + col) * KP + s * 32 + hi * 8]);
#pragma unroll
        for (int u = 0; u < QT; ++u)
          s4[u][pt] = mfma_bf16(a, qf[u][s], s4[u][pt]);
      }
    }
    const bool edge = pg * PG + PG - 1 > p0 + w0; // uniform over the wave
    bf16x8_v pf[QT][2];
#pragma unroll
    for (int u = 0; u < QT; ++u) {
      const int qpos = p0 + w0 + u * 16 + col;
      float mx = NEG_BIG;
#pragma unroll
      for (int pt = 0; pt < 4; ++pt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          float v = s4[u][pt][r] * scale2;
          if (edge) {
            const int p = pg * PG + pt * 16 + hi * 4 + r;
            v = p <= qpos && p <= last ? v : NEG_BIG;
          }
          s4[u][pt][r] = v;
          mx = fmaxf(mx, v);
        }
      mx = fmaxf(mx, __shfl_xor(mx, 16, QSA_WAVE));
      mx = fmaxf(mx, __shfl_xor(mx, 32, QSA_WAVE));
      const float mn = fmaxf(m[u], mx);
      const float alpha = exp2_hw(m[u] - mn);     // page 0 shows every row a
                                                  // key: mn is finite
      m[u] = mn;
      float psum = 0.f;
      uint2 pk[4];
#pragma unroll
      for (int pt = 0; pt < 4; ++pt) {
        float p[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          p[r] = exp2_hw(s4[u][pt][r] - mn);
          psum += p[r];
        }
        pk[pt] = make_uint2(cvt_bf16x2(p[0], p[1]), cvt_bf16x2(p[2], p[3]));
      }
#pragma unroll
      for (int s = 0; s < 2; ++s)
        pf[u][s] = __builtin_bit_cast(
            bf16x8_v, make_uint4(pk[2 * s].x, pk[2 * s].y, pk[2 * s + 1].x,
                                 pk[2 * s + 1].y));
      l[u] = l[u] * alpha + psum;
#pragma unroll
      for (int t = 0; t < ET; ++t) acc[u][t] *= alpha;
    }
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int t = 0; t < ET; ++t) {
        const bf16x8_v a =
            lds_frag_tr(vt, VP, s * 32, s * 32 + 16, t * 16, lane);
#pragma unroll
        for (int u = 0; u < QT; ++u)
          acc[u][t] = mfma_bf16(a, pf[u][s], acc[u][t]);
      }
  }
  const float sk = sink ? sink[h] * LOG2E : NEG_BIG;
#pragma unroll
  for (int u = 0; u < QT; ++u) {
    l[u] += __shfl_xor(l[u], 16, QSA_WAVE);
    l[u] += __shfl_xor(l[u], 32, QSA_WAVE);
    const float top = fmaxf(m[u], sk);
    const float f = m[u] > NEG_BIG ? exp2f(m[u] - top) : 0.f;
    const float den = l[u] * f + (sink ? exp2f(sk - top) : 0.f);
    const float inv = den > 0.f ? f / den * out_scale : 0.f;
    const int i = w0 + u * 16 + col;
    if (i < n) {
      const bf16_t* gr = gate + (long long)(r0 + i) * gstride +
                         (long long)h * E;
      bf16_t* orow = out + (long long)(r0 + i) * ostride + (long long)h * E;
#pragma unroll
      for (int t = 0; t < ET; ++t) {
        const int e = t * 16 + hi * 4;
        if (e < E) {                              // E % 8 == 0
          float o[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) o[r] = acc[u][t][r] * inv;
          if (gate) {
            float gv[4];
            ldv<bf16_t, 4>(gr + e, gv);
#pragma unroll
            for (int r = 0; r < 4; ++r) o[r] /= 1.f + __expf(-gv[r]);
          }
          stv<bf16_t, 4>(orow + e, o);
        }
      }
    }
  }
}

extern "C" void qsa_gqa_portions_launch(
    const bf16_t* q, const bf16_t* kc, const bf16_t* vc,
    const int* block_table, int max_pages, const float* sink,
    const bf16_t* gate, long long gstride, const int* qb_item,
    const int* qb_t0, const int* off, const int* start, const int* len,
    bf16_t* out, long long ostride, int QB, int H, int G, int D, int E,
    float scale, float out_scale, int wide, hipStream_t st) {
  dim3 grid((unsigned)((long long)QB * H));
  const float scale2 = scale * LOG2E;
#define QSA_GP(K, V, Q)                                                      \
  hipLaunchKernelGGL((qsa_gqa_portions<K, V, Q>), grid, dim3(256), 0, st, q, \
                     kc, vc, block_table, max_pages, sink, gate, gstride,    \
                     qb_item, qb_t0, off, start, len, out, ostride, H, G, D, \
                     E, scale2, out_scale)
#define QSA_GP_E(K, W)                                                       \
  if (E <= 32) { if (W) QSA_GP(K, 2, 2); else QSA_GP(K, 2, 1); }             \
  else if (E <= 64) { if (W) QSA_GP(K, 4, 2); else QSA_GP(K, 4, 1); }        \
  else if (E <= 128) { if (W) QSA_GP(K, 8, 2); else QSA_GP(K, 8, 1); }       \
  else QSA_GP(K, 16, 1)
  if (D <= 32) { QSA_GP_E(1, wide); }
  else if (D <= 64) { QSA_GP_E(2, wide); }
  else if (D <= 128) { QSA_GP_E(4, wide); }
  else if (E <= 128) { if (E <= 32) QSA_GP(8, 2, 1);
                       else if (E <= 64) QSA_GP(8, 4, 1);
                       else QSA_GP(8, 8, 1); }
  else { QSA_GP(8, 16, 1); }
#undef QSA_GP_E
#undef QSA_GP
}
