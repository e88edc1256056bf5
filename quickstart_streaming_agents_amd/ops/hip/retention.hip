// Retention (linear attention with one fixed decay per head) for gfx950.
//
//   S_t = decay * S_(t-1) + k_t v_t^T        S [dim, vdim], f32
//   o_t = S_t^T q_t,  out = o / rms(o) * silu(gate)
//
// with q, k rotated (first `rot` dims, pairs i / i + rot/2) and k scaled
// after the rotation.  Operands sit side by side in one projection row
// [q | k | v | gate].  State: [slots, H, dim, vdim] f32, one slot per live
// sequence.  A sequence's state is taken as zero at position 0, so slots
// need no clearing between owners.
//
// Kernels
//   qsa_retention_decode   one token per row: rotate, update, read-out, norm
//                          and gate in one pass over the state (HBM-bound).
//   qsa_retention_seq      token loop per (portion, head), any size and
//                          storage type; the f32 path.
//   chunked prefill (bf16 storage, matrix cores), chunks of 64 tokens:
//     qsa_retention_rotate   rotated q, k as bf16 hi/lo planes, zero-padded
//     qsa_retention_state    walks the chunks of a portion, state tile in
//                            accumulators; leaves the state before each
//                            chunk as hi/lo planes [chunk, H, vdim, dim]
//     qsa_retention_out      per (chunk, head): inter-chunk read-out,
//                            intra-chunk masked product, norm, gate
// Every operand that f32 rounding matters for is a hi/lo pair, so the
// chunked result agrees with the token loop to ~2^-16; v is bf16 already.
#include "lm_common.h"

#define RC 64  // tokens per chunk

// ---------------------------------------------------------------------------
// Shared scalar pieces
// ---------------------------------------------------------------------------
// element d of a rotated head vector
template <typename T>
__device__ __forceinline__ float rot_elem(const T* x, int d, int rot,
                                          const float* cs, const float* sn) {
  const float a = ldf<T>(x + d);
  const int half = rot >> 1;
  if (d < half) return a * cs[d] - ldf<T>(x + d + half) * sn[d];
  if (d < rot) return a * cs[d - half] + ldf<T>(x + d - half) * sn[d - half];
  return a;
}

// ---------------------------------------------------------------------------
// Decode: one block per (row, head).
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__global__ void __launch_bounds__(512)
qsa_retention_decode(const T* __restrict__ x, long long xstride,
                     const float* __restrict__ cos_t,
                     const float* __restrict__ sin_t,
                     const float* __restrict__ decay, float* __restrict__ state,
                     const int* __restrict__ slots,
                     const int* __restrict__ seq_lens, T* __restrict__ out,
                     int H, int D, int E, int rot, int CW, float kscale,
                     float eps, int table_len) {
  extern __shared__ float sm[];
  float* qs = sm;                 // D
  float* ks = qs + D;             // D
  float* os = ks + D;             // E
  float* red = os + (E + 3) / 4 * 4;  // threads * VEC
  __shared__ float scratch[8];
  const int b = blockIdx.x / H, h = blockIdx.x % H;
  const int tid = threadIdx.x, nth = blockDim.x;
  const int pos = seq_lens[b] - 1;
  const int slot = slots[b];
  T* orow = out + ((long long)b * H + h) * E;
  if (pos < 0 || slot < 0 || pos >= table_len) {   // uniform over the block
    for (int e = tid; e < E; e += nth) stf<T>(orow + e, 0.f);
    return;
  }
  const T* q = x + (long long)b * xstride + (long long)h * D;
  const T* k = x + (long long)b * xstride + (long long)(H + h) * D;
  const T* v = x + (long long)b * xstride + 2LL * H * D + (long long)h * E;
  const T* g = v + (long long)H * E;
  const float* cs = cos_t + (long long)pos * (rot >> 1);
  const float* sn = sin_t + (long long)pos * (rot >> 1);
  for (int d = tid; d < D; d += nth) {
    qs[d] = rot_elem<T>(q, d, rot, cs, sn);
    ks[d] = rot_elem<T>(k, d, rot, cs, sn) * kscale;
  }
  __syncthreads();
  const float dec = decay[h];
  const bool fresh = pos == 0;
  float* S = state + ((long long)slot * H + h) * D * E;
  const int G = nth / CW;          // dim groups
  const int c0 = tid % CW, g0 = tid / CW;
  const int NV = E / VEC;
  float ss = 0.f;
  for (int cb = 0; cb < NV; cb += CW) {
    const int c = cb + c0;
    float acc[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) acc[j] = 0.f;
    if (c < NV) {
      float vv[VEC];
      ldv<T, VEC>(v + c * VEC, vv);
      float* sp = S + c * VEC;
#pragma unroll 4
      for (int d = g0; d < D; d += G) {
        float s[VEC];
        if (fresh) {
#pragma unroll
          for (int j = 0; j < VEC; ++j) s[j] = 0.f;
        } else {
          ldv<float, VEC>(sp + (long long)d * E, s);
        }
        const float kd = ks[d], qd = qs[d];
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          s[j] = fmaf(dec, s[j], kd * vv[j]);
          acc[j] = fmaf(qd, s[j], acc[j]);
        }
        stv<float, VEC>(sp + (long long)d * E, s);
      }
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) red[tid * VEC + j] = acc[j];
    __syncthreads();
    if (g0 == 0 && c < NV) {
      for (int gg = 1; gg < G; ++gg)
#pragma unroll
        for (int j = 0; j < VEC; ++j) acc[j] += red[(gg * CW + c0) * VEC + j];
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        os[c * VEC + j] = acc[j];
        ss = fmaf(acc[j], acc[j], ss);
      }
    }
    __syncthreads();
  }
  ss = block_reduce_sum(ss, scratch);
  const float inv = 1.f / sqrtf(ss / (float)E + eps);
  for (int e = tid; e < E; e += nth)
    stf<T>(orow + e, os[e] * inv * silu_f(ldf<T>(g + e)));
}

extern "C" void qsa_retention_decode_launch(
    const void* x, long long xstride, const float* cos_t, const float* sin_t,
    const float* decay, float* state, const int* slots, const int* seq_lens,
    void* out, int B, int H, int D, int E, int rot, float kscale, float eps,
    int table_len, int f32, int vec4, hipStream_t st) {
  const int nv = vec4 ? E / 4 : E;
  int cw = 1;
  while (cw < nv && cw < 256) cw <<= 1;
  const int threads = 256;
  const size_t lds = sizeof(float) *
      (2 * (size_t)D + (E + 3) / 4 * 4 + threads * (vec4 ? 4 : 1));
#define QSA_RD(T, V)                                                         \
  hipLaunchKernelGGL((qsa_retention_decode<T, V>), dim3((unsigned)(B * H)),  \
                     dim3(threads), lds, st, (const T*)x, xstride, cos_t,    \
                     sin_t, decay, state, slots, seq_lens, (T*)out, H, D, E, \
                     rot, cw, kscale, eps, table_len)
  if (f32) { if (vec4) QSA_RD(float, 4); else QSA_RD(float, 1); }
  else     { if (vec4) QSA_RD(bf16_t, 4); else QSA_RD(bf16_t, 1); }
#undef QSA_RD
}

// ---------------------------------------------------------------------------
// Token loop over a portion: one block per (portion, head), thread t owns
// columns t, t + 256, ...; the state tile stays in LDS when it fits.
// ---------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256)
qsa_retention_seq(const T* __restrict__ x, long long xstride,
                  const float* __restrict__ cos_t,
                  const float* __restrict__ sin_t,
                  const float* __restrict__ decay, float* __restrict__ state,
                  const int* __restrict__ slots, const int* __restrict__ off,
                  const int* __restrict__ start, const int* __restrict__ len,
                  T* __restrict__ out, int H, int D, int E, int rot,
                  float kscale, float eps, int table_len, int in_lds) {
  extern __shared__ float sm[];
  float* qs = sm;
  float* ks = qs + D;
  float* os = ks + D;
  float* tile = os + E;
  __shared__ float scratch[8];
  const int it = blockIdx.x / H, h = blockIdx.x % H;
  const int tid = threadIdx.x, nth = blockDim.x;
  const int n = len[it], p0 = start[it], r0 = off[it], slot = slots[it];
  if (slot < 0) return;
  const float dec = decay[h];
  float* Sg = state + ((long long)slot * H + h) * D * E;
  float* S = in_lds ? tile : Sg;
  for (int i = tid; i < D * E; i += nth)
    if (p0 == 0) S[i] = 0.f;
    else if (in_lds) S[i] = Sg[i];
  for (int t = 0; t < n; ++t) {
    const T* xr = x + (long long)(r0 + t) * xstride;
    const T* q = xr + (long long)h * D;
    const T* k = xr + (long long)(H + h) * D;
    const T* v = xr + 2LL * H * D + (long long)h * E;
    const T* g = v + (long long)H * E;
    int p = p0 + t;
    p = p < table_len ? p : table_len - 1;
    const float* cs = cos_t + (long long)p * (rot >> 1);
    const float* sn = sin_t + (long long)p * (rot >> 1);
    __syncthreads();   // previous token's readers of qs/ks/os are done
    for (int d = tid; d < D; d += nth) {
      qs[d] = rot_elem<T>(q, d, rot, cs, sn);
      ks[d] = rot_elem<T>(k, d, rot, cs, sn) * kscale;
    }
    __syncthreads();
    float ss = 0.f;
    for (int e = tid; e < E; e += nth) {
      const float ve = ldf<T>(v + e);
      float acc = 0.f;
      for (int d = 0; d < D; ++d) {
        const float s = fmaf(dec, S[d * E + e], ks[d] * ve);
        S[d * E + e] = s;
        acc = fmaf(qs[d], s, acc);
      }
      os[e] = acc;
      ss = fmaf(acc, acc, ss);
    }
    ss = block_reduce_sum(ss, scratch);
    const float inv = 1.f / sqrtf(ss / (float)E + eps);
    T* orow = out + ((long long)(r0 + t) * H + h) * E;
    for (int e = tid; e < E; e += nth)
      stf<T>(orow + e, os[e] * inv * silu_f(ldf<T>(g + e)));
  }
  if (in_lds) {
    __syncthreads();
    for (int i = tid; i < D * E; i += nth) Sg[i] = S[i];
  }
}

extern "C" void qsa_retention_seq_launch(
    const void* x, long long xstride, const float* cos_t, const float* sin_t,
    const float* decay, float* state, const int* slots, const int* off,
    const int* start, const int* len, void* out, int n_items, int H, int D,
    int E, int rot, float kscale, float eps, int table_len, int f32,
    hipStream_t st) {
  size_t lds = sizeof(float) * (2 * (size_t)D + E);
  const size_t with_tile = lds + sizeof(float) * (size_t)D * E;
  const int in_lds = with_tile <= 60 * 1024;
  if (in_lds) lds = with_tile;
#define QSA_RS(T)                                                           \
  hipLaunchKernelGGL((qsa_retention_seq<T>), dim3((unsigned)(n_items * H)), \
                     dim3(256), lds, st, (const T*)x, xstride, cos_t,       \
                     sin_t, decay, state, slots, off, start, len, (T*)out,  \
                     H, D, E, rot, kscale, eps, table_len, in_lds)
  if (f32) QSA_RS(float); else QSA_RS(bf16_t);
#undef QSA_RS
}

// ---------------------------------------------------------------------------
// Chunked prefill, step 1: planes[p][row][h][DP], p = q.hi, q.lo, k.hi, k.lo
// ---------------------------------------------------------------------------
__global__ void __launch_bounds__(256)
qsa_retention_rotate(const bf16_t* __restrict__ x, long long xstride,
                     const float* __restrict__ cos_t,
                     const float* __restrict__ sin_t,
                     const int* __restrict__ positions,
                     bf16_t* __restrict__ planes, long long rows, int H,
                     int D, int DP, int rot, float kscale, int table_len) {
  const long long plane = rows * H * DP;
  const long long n = rows * H * (DP / 4);
  for (long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x; i < n;
       i += (long long)gridDim.x * blockDim.x) {
    const int d0 = (int)(i % (DP / 4)) * 4;
    const long long rh = i / (DP / 4);
    const int h = (int)(rh % H);
    const long long row = rh / H;
    int p = positions[row];
    p = p < table_len ? p : table_len - 1;
    const float* cs = cos_t + (long long)p * (rot >> 1);
    const float* sn = sin_t + (long long)p * (rot >> 1);
    const bf16_t* q = x + row * xstride + (long long)h * D;
    const bf16_t* k = q + (long long)H * D;
    float qv[4], kv[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int d = d0 + j;
      qv[j] = d < D ? rot_elem<bf16_t>(q, d, rot, cs, sn) : 0.f;
      kv[j] = d < D ? rot_elem<bf16_t>(k, d, rot, cs, sn) * kscale : 0.f;
    }
    uint2 a, b;
    bf16_t* o = planes + rh * DP + d0;
    split4_bf16(qv[0], qv[1], qv[2], qv[3], a, b);
    *reinterpret_cast<uint2*>(o) = a;
    *reinterpret_cast<uint2*>(o + plane) = b;
    split4_bf16(kv[0], kv[1], kv[2], kv[3], a, b);
    *reinterpret_cast<uint2*>(o + 2 * plane) = a;
    *reinterpret_cast<uint2*>(o + 3 * plane) = b;
  }
}

extern "C" void qsa_retention_rotate_launch(
    const bf16_t* x, long long xstride, const float* cos_t,
    const float* sin_t, const int* positions, bf16_t* planes, long long rows,
    int H, int D, int DP, int rot, float kscale, int table_len,
    hipStream_t st) {
  const long long n = rows * H * (DP / 4);
  const long long want = (n + 255) / 256;
  hipLaunchKernelGGL(qsa_retention_rotate,
                     dim3((unsigned)(want > 32768 ? 32768 : want)), dim3(256),
                     0, st, x, xstride, cos_t, sin_t, positions, planes, rows,
                     H, D, DP, rot, kscale, table_len);
}

// ---------------------------------------------------------------------------
// Step 2: state walk.  Block = (portion, head, 64 value columns); wave w owns
// 16 of the columns and all DP rows of the state tile in accumulators.
//   S_(c+1) = decay^n S_c + sum_j k_j (decay^(n-1-j) v_j)^T
// ---------------------------------------------------------------------------
template <int KS>  // DP = 32 * KS
__global__ void __launch_bounds__(256)
qsa_retention_state(const bf16_t* __restrict__ x, long long xstride,
                    long long voff, const bf16_t* __restrict__ planes,
                    long long rows, const float* __restrict__ log2_decay,
                    float* __restrict__ state, const int* __restrict__ slots,
                    const int* __restrict__ off, const int* __restrict__ start,
                    const int* __restrict__ len,
                    const int* __restrict__ chunk0,
                    bf16_t* __restrict__ prefix, long long n_chunks, int H,
                    int D, int E, int EP) {
  constexpr int DP = 32 * KS;
  constexpr int KP = DP + 16;       // LDS pitches (elements)
  constexpr int VP = 64 + 16;
  constexpr int KLD = RC * DP / 8 / 256;   // 16 B groups per thread and plane
  __shared__ __attribute__((aligned(16))) bf16_t kt[2][RC * KP];
  __shared__ __attribute__((aligned(16))) bf16_t vt[2][RC * VP];
  const int VT = (EP + 63) / 64;
  const int vtile = blockIdx.x % VT;
  const int h = (blockIdx.x / VT) % H;
  const int it = blockIdx.x / (VT * H);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int col = lane & 15, hi = lane >> 4;
  const int n = len[it], p0 = start[it], r0 = off[it], slot = slots[it];
  const float l2d = log2_decay[h];
  const int v0 = vtile * 64;
  const int e = v0 + wave * 16 + col;          // this lane's value column
  float* S = state + ((long long)slot * H + h) * D * E;
  const long long plane = rows * H * DP;
  const bf16_t* kpl = planes + 2 * plane;

  f32x4_v acc[2 * KS];
#pragma unroll
  for (int t = 0; t < 2 * KS; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = t * 16 + hi * 4 + r;
      acc[t][r] = (p0 > 0 && d < D && e < E) ? S[(long long)d * E + e] : 0.f;
    }

  u32x4_v kh[KLD], kl[KLD], vreg[2];
#define QSA_FETCH(t0_)                                                        \
  {                                                                           \
    _Pragma("unroll") for (int u = 0; u < KLD; ++u) {                         \
      const int g = tid + u * 256;                                            \
      const int tr = min((t0_) + g / (DP / 8), n - 1);                        \
      const bf16_t* src = kpl + ((long long)(r0 + tr) * H + h) * DP +         \
                          (g % (DP / 8)) * 8;                                 \
      kh[u] = *reinterpret_cast<const u32x4_v*>(src);                           \
      kl[u] = *reinterpret_cast<const u32x4_v*>(src + plane);                   \
    }                                                                         \
    _Pragma("unroll") for (int u = 0; u < 2; ++u) {                           \
      const int g = tid + u * 256;                                            \
      const int tr = min((t0_) + (g >> 3), n - 1);                            \
      const int cc = min(v0 + (g & 7) * 8, E - 8); /* E % 8 == 0 */           \
      vreg[u] = *reinterpret_cast<const u32x4_v*>(                              \
          x + (long long)(r0 + tr) * xstride + voff + (long long)h * E + cc); \
    }                                                                         \
  }
  QSA_FETCH(0)
  const int nc = (n + RC - 1) / RC;
  for (int c = 0; c < nc; ++c) {
    const int t0 = c * RC;
    const int m = min(RC, n - t0);
    __syncthreads();                 // previous chunk's LDS readers are done
#pragma unroll
    for (int u = 0; u < KLD; ++u) {
      const int g = tid + u * 256;
      const int o = g / (DP / 8) * KP + (g % (DP / 8)) * 8;
      *reinterpret_cast<u32x4_v*>(&kt[0][o]) = kh[u];
      *reinterpret_cast<u32x4_v*>(&kt[1][o]) = kl[u];
    }
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int g = tid + u * 256;
      const int row = g >> 3, cc = (g & 7) * 8;
      const bool ok = row < m && v0 + cc < E;
      const float f = exp2f((float)(m - 1 - row) * l2d);
      const u32x4_v pk = ok ? vreg[u] : (u32x4_v){0, 0, 0, 0};
      const float fo = ok ? f : 0.f;
      const float2 v01 = bf16x2_to_f32x2(pk.x), v23 = bf16x2_to_f32x2(pk.y);
      const float2 v45 = bf16x2_to_f32x2(pk.z), v67 = bf16x2_to_f32x2(pk.w);
      uint2 h0, l0, h1, l1;
      split4_bf16(v01.x * fo, v01.y * fo, v23.x * fo, v23.y * fo, h0, l0);
      split4_bf16(v45.x * fo, v45.y * fo, v67.x * fo, v67.y * fo, h1, l1);
      *reinterpret_cast<uint4*>(&vt[0][row * VP + cc]) =
          make_uint4(h0.x, h0.y, h1.x, h1.y);
      *reinterpret_cast<uint4*>(&vt[1][row * VP + cc]) =
          make_uint4(l0.x, l0.y, l1.x, l1.y);
    }
    __syncthreads();
    if (c + 1 < nc) QSA_FETCH(t0 + RC)

    // state before this chunk (nothing precedes the first token)
    if ((c > 0 || p0 > 0) && e < EP) {
      bf16_t* ph = prefix +
          (((long long)(chunk0[it] + c) * H + h) * EP + e) * DP;
      bf16_t* pl = ph + n_chunks * H * EP * DP;
#pragma unroll
      for (int t = 0; t < 2 * KS; ++t) {
        uint2 a, b;
        split4_bf16(acc[t][0], acc[t][1], acc[t][2], acc[t][3], a, b);
        const int d = t * 16 + hi * 4;
        *reinterpret_cast<uint2*>(ph + d) = a;
        *reinterpret_cast<uint2*>(pl + d) = b;
      }
    }
    const float dn = exp2f((float)m * l2d);
#pragma unroll
    for (int t = 0; t < 2 * KS; ++t) acc[t] *= dn;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const bf16x8_v bh =
          lds_frag_tr(vt[0], VP, s * 32, s * 32 + 16, wave * 16, lane);
      const bf16x8_v bl =
          lds_frag_tr(vt[1], VP, s * 32, s * 32 + 16, wave * 16, lane);
#pragma unroll
      for (int t = 0; t < 2 * KS; ++t) {
        const bf16x8_v ah =
            lds_frag_tr(kt[0], KP, s * 32, s * 32 + 16, t * 16, lane);
        const bf16x8_v al =
            lds_frag_tr(kt[1], KP, s * 32, s * 32 + 16, t * 16, lane);
        acc[t] = mfma_bf16(ah, bh, acc[t]);
        acc[t] = mfma_bf16(ah, bl, acc[t]);
        acc[t] = mfma_bf16(al, bh, acc[t]);
      }
    }
  }
#pragma unroll
  for (int t = 0; t < 2 * KS; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = t * 16 + hi * 4 + r;
      if (d < D && e < E) S[(long long)d * E + e] = acc[t][r];
    }
}

#undef QSA_FETCH

extern "C" void qsa_retention_state_launch(
    const bf16_t* x, long long xstride, long long voff, const bf16_t* planes,
    long long rows, const float* log2_decay, float* state, const int* slots,
    const int* off, const int* start, const int* len, const int* chunk0,
    bf16_t* prefix, long long n_chunks, int n_items, int H, int D, int DP,
    int E, int EP, hipStream_t st) {
  dim3 grid((unsigned)(n_items * H * ((EP + 63) / 64)));
#define QSA_ST(K)                                                           \
  case K:                                                                   \
    hipLaunchKernelGGL((qsa_retention_state<K>), grid, dim3(256), 0, st, x, \
                       xstride, voff, planes, rows, log2_decay, state,      \
                       slots, off, start, len, chunk0, prefix, n_chunks, H, \
                       D, E, EP);                                           \
    break;
  switch (DP / 32) { QSA_ST(1) QSA_ST(2) QSA_ST(4) QSA_ST(8) }
#undef QSA_ST
}

// ---------------------------------------------------------------------------
// Step 3: outputs of one (chunk, head).  Wave w owns rows 16w..16w+15 and all
// value columns, with O^T in accumulators (row = value, column = token):
//   O^T  = decay^(i+1) * (S^T q_i)  +  V^T P^T,   P_ij = q_i.k_j decay^(i-j)
// P^T leaves the first product in exactly the operand layout of the second
// one (the order of the summed index is free), so nothing is shuffled.
// ---------------------------------------------------------------------------
template <int KS, int ET>  // DP = 32*KS, up to 16*ET value columns
__global__ void __launch_bounds__(256)
qsa_retention_out(const bf16_t* __restrict__ x, long long xstride,
                  long long voff, const bf16_t* __restrict__ planes,
                  long long rows, const float* __restrict__ log2_decay,
                  const int* __restrict__ off, const int* __restrict__ start,
                  const int* __restrict__ len,
                  const int* __restrict__ chunk_item,
                  const int* __restrict__ chunk_t0,
                  const bf16_t* __restrict__ prefix, long long n_chunks,
                  bf16_t* __restrict__ out, int H, int E, int EP, float eps) {
  constexpr int DP = 32 * KS;
  constexpr int KP = DP + 8;
  constexpr int VP = 16 * ET + 16;
  __shared__ __attribute__((aligned(16))) bf16_t kt[2][RC * KP];
  __shared__ __attribute__((aligned(16))) bf16_t vt[RC * VP];
  const int h = blockIdx.x % H;
  const int ch = blockIdx.x / H;
  const int it = chunk_item[ch], t0 = chunk_t0[ch];
  const int m = min(RC, len[it] - t0);
  const long long r0 = off[it] + t0;
  const bool has_prefix = t0 > 0 || start[it] > 0;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int col = lane & 15, hi = lane >> 4;
  const float l2d = log2_decay[h];
  const long long plane = rows * H * DP;

  // stage k planes and v
#pragma unroll
  for (int p = 0; p < 2; ++p)
    for (int g = tid; g < RC * DP / 8; g += 256) {
      const int row = g / (DP / 8), c = (g % (DP / 8)) * 8;
      *reinterpret_cast<uint4*>(&kt[p][row * KP + c]) =
          *reinterpret_cast<const uint4*>(
              planes + (2 + p) * plane +
              ((r0 + min(row, m - 1)) * H + h) * DP + c);
    }
  const int EG = (EP + 7) / 8;
  for (int g = tid; g < RC * EG; g += 256) {
    const int row = g / EG, c = (g % EG) * 8;
    uint4 v = make_uint4(0, 0, 0, 0);
    if (row < m && c < E)
      v = *reinterpret_cast<const uint4*>(
          x + (r0 + row) * xstride + voff + (long long)h * E + c);
    *reinterpret_cast<uint4*>(&vt[row * VP + c]) = v;
  }
  // this lane's token row i and its query operands
  const int i = wave * 16 + col;
  const long long qrow = r0 + min(i, m - 1);
  bf16x8_v qh[KS], ql[KS];
#pragma unroll
  for (int s = 0; s < KS; ++s) {
    const long long o = (qrow * H + h) * DP + s * 32 + hi * 8;
    qh[s] = *reinterpret_cast<const bf16x8_v*>(planes + o);
    ql[s] = *reinterpret_cast<const bf16x8_v*>(planes + plane + o);
  }
  f32x4_v acc[ET];
#pragma unroll
  for (int t = 0; t < ET; ++t) acc[t] = (f32x4_v){0.f, 0.f, 0.f, 0.f};

  if (has_prefix) {                                   // uniform
    const bf16_t* ph = prefix + ((long long)ch * H + h) * EP * DP;
    const bf16_t* pl = ph + n_chunks * H * EP * DP;
#pragma unroll
    for (int t = 0; t < ET; ++t) {
      if (t * 16 >= EP) break;                        // uniform
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const int o = (t * 16 + col) * DP + s * 32 + hi * 8;
        const bf16x8_v ah = *reinterpret_cast<const bf16x8_v*>(ph + o);
        const bf16x8_v al = *reinterpret_cast<const bf16x8_v*>(pl + o);
        acc[t] = mfma_bf16(ah, qh[s], acc[t]);
        acc[t] = mfma_bf16(ah, ql[s], acc[t]);
        acc[t] = mfma_bf16(al, qh[s], acc[t]);
      }
    }
    const float f = exp2f((float)(i + 1) * l2d);
#pragma unroll
    for (int t = 0; t < ET; ++t) acc[t] *= f;
  }
  __syncthreads();

  // keys up to this wave's last row, 32 at a time
  const int pairs = (wave >> 1) + 1;
  for (int s2 = 0; s2 < pairs; ++s2) {
    bf16x8_v pbh, pbl;
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int pt = s2 * 2 + u;
      f32x4_v sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const int o = (pt * 16 + col) * KP + s * 32 + hi * 8;
        const bf16x8_v ah = *reinterpret_cast<const bf16x8_v*>(&kt[0][o]);
        const bf16x8_v al = *reinterpret_cast<const bf16x8_v*>(&kt[1][o]);
        sc = mfma_bf16(ah, qh[s], sc);
        sc = mfma_bf16(ah, ql[s], sc);
        sc = mfma_bf16(al, qh[s], sc);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = pt * 16 + hi * 4 + r;
        const float f = (j <= i && j < m) ? exp2f((float)(i - j) * l2d) : 0.f;
        bf16_t a, b;
        split_bf16(j <= i && j < m ? sc[r] * f : 0.f, a, b);
        pbh[u * 4 + r] = (short)a;
        pbl[u * 4 + r] = (short)b;
      }
    }
#pragma unroll
    for (int t = 0; t < ET; ++t) {
      if (t * 16 >= EP) break;
      const bf16x8_v av =
          lds_frag_tr(vt, VP, s2 * 32, s2 * 32 + 16, t * 16, lane);
      acc[t] = mfma_bf16(av, pbh, acc[t]);
      acc[t] = mfma_bf16(av, pbl, acc[t]);
    }
  }

  // per-token rms over the value columns, gate, store
  float ss = 0.f;
#pragma unroll
  for (int t = 0; t < ET; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) ss = fmaf(acc[t][r], acc[t][r], ss);
  ss += __shfl_xor(ss, 16, QSA_WAVE);
  ss += __shfl_xor(ss, 32, QSA_WAVE);
  const float inv = 1.f / sqrtf(ss / (float)E + eps);
  if (i < m) {
    const bf16_t* g = x + (r0 + i) * xstride + voff + (long long)H * E +
                      (long long)h * E;
    bf16_t* orow = out + ((r0 + i) * H + h) * E;
#pragma unroll
    for (int t = 0; t < ET; ++t) {
      const int e0 = t * 16 + hi * 4;
      if (e0 < E) {                                   // E % 8 == 0
        float gv[4], o[4];
        ldv<bf16_t, 4>(g + e0, gv);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          o[r] = acc[t][r] * inv * (gv[r] / (1.f + __expf(-gv[r])));
        stv<bf16_t, 4>(orow + e0, o);
      }
    }
  }
}

extern "C" void qsa_retention_out_launch(
    const bf16_t* x, long long xstride, long long voff, const bf16_t* planes,
    long long rows, const float* log2_decay, const int* off,
    const int* start, const int* len, const int* chunk_item,
    const int* chunk_t0, const bf16_t* prefix, long long n_chunks,
    bf16_t* out, int H, int DP, int E, int EP, float eps, hipStream_t st) {
  dim3 grid((unsigned)(n_chunks * H));
#define QSA_RO(K, V)                                                        \
  hipLaunchKernelGGL((qsa_retention_out<K, V>), grid, dim3(256), 0, st, x,  \
                     xstride, voff, planes, rows, log2_decay, off, start,   \
                     len, chunk_item, chunk_t0, prefix, n_chunks, out, H,   \
                     E, EP, eps)
#define QSA_RO_E(K)                                                         \
  if (EP <= 32) QSA_RO(K, 2);                                               \
  else if (EP <= 64) QSA_RO(K, 4);                                          \
  else if (EP <= 128) QSA_RO(K, 8);                                         \
  else if (EP <= 256) QSA_RO(K, 16);                                        \
  else QSA_RO(K, 32)
  switch (DP / 32) {
    case 1: QSA_RO_E(1); break;
    case 2: QSA_RO_E(2); break;
    case 4: QSA_RO_E(4); break;
    case 8: QSA_RO_E(8); break;
  }
#undef QSA_RO_E
#undef QSA_RO
}
