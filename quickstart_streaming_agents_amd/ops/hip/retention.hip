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
//                            chunk as hi/lo matrix-core operands
//     qsa_retention_out      per (chunk, head): inter-chunk read-out,
//                            intra-chunk masked product, norm, gate
// Every rounded operand is a bf16 hi/lo pair on the matrix cores (q, k, the
// decayed v, the state, the intra-chunk weights), so the chunked result agrees
// with the token loop to ~2^-16; v is bf16 already.  One-sided rounding would
// show: the norm over a head blows it up where S^T q is small.
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
__global__ void __launch_bounds__(1024)
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
  __shared__ float scratch[16];
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
  // few blocks: wide ones, so that enough of the state is in flight
  const int threads =
      (long long)B * H <= 512 && (long long)D * E >= 16384 ? 1024 : 256;
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
// One thread per 8 dims of a head of a row, q and k.  FAST: whole groups on
// either side of the rotation pairs (rot % 16 == 0, D % 8 == 0, 16 B rows).
template <bool FAST>
__global__ void __launch_bounds__(256)
qsa_retention_rotate(const bf16_t* __restrict__ x, long long xstride,
                     const float* __restrict__ cos_t,
                     const float* __restrict__ sin_t,
                     const int* __restrict__ positions,
                     bf16_t* __restrict__ planes, long long rows, int H,
                     int D, int DP, int rot, float kscale, int table_len) {
  const long long plane = rows * H * DP;
  const int per_row = H * (DP / 8);
  const long long row = blockIdx.x;
  const int half = rot >> 1;
  int p = positions[row];
  p = p < table_len ? p : table_len - 1;
  const float* cs = cos_t + (long long)p * half;
  const float* sn = sin_t + (long long)p * half;
  for (int g = threadIdx.x; g < per_row; g += blockDim.x) {
    const int h = g / (DP / 8), d0 = (g % (DP / 8)) * 8;
    const bf16_t* q = x + row * xstride + (long long)h * D;
    const bf16_t* k = q + (long long)H * D;
    float qv[8], kv[8];
    if (FAST) {
      if (d0 < D) {
        ldv<bf16_t, 8>(q + d0, qv);
        ldv<bf16_t, 8>(k + d0, kv);
        if (d0 < rot) {
          const bool lo = d0 < half;
          const int o = lo ? d0 + half : d0 - half, c = lo ? d0 : d0 - half;
          float qo[8], ko[8], cc[8], ss[8];
          ldv<bf16_t, 8>(q + o, qo);
          ldv<bf16_t, 8>(k + o, ko);
          ldv<float, 8>(cs + c, cc);
          ldv<float, 8>(sn + c, ss);
          const float sg = lo ? -1.f : 1.f;
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            qv[j] = qv[j] * cc[j] + sg * qo[j] * ss[j];
            kv[j] = kv[j] * cc[j] + sg * ko[j] * ss[j];
          }
        }
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) qv[j] = kv[j] = 0.f;
      }
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int d = d0 + j;
        qv[j] = d < D ? rot_elem<bf16_t>(q, d, rot, cs, sn) : 0.f;
        kv[j] = d < D ? rot_elem<bf16_t>(k, d, rot, cs, sn) : 0.f;
      }
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) kv[j] *= kscale;
    uint2 a0, b0, a1, b1;
    bf16_t* o = planes + (row * H + h) * DP + d0;
    split4_bf16(qv[0], qv[1], qv[2], qv[3], a0, b0);
    split4_bf16(qv[4], qv[5], qv[6], qv[7], a1, b1);
    *reinterpret_cast<uint4*>(o) = make_uint4(a0.x, a0.y, a1.x, a1.y);
    *reinterpret_cast<uint4*>(o + plane) = make_uint4(b0.x, b0.y, b1.x, b1.y);
    split4_bf16(kv[0], kv[1], kv[2], kv[3], a0, b0);
    split4_bf16(kv[4], kv[5], kv[6], kv[7], a1, b1);
    *reinterpret_cast<uint4*>(o + 2 * plane) =
        make_uint4(a0.x, a0.y, a1.x, a1.y);
    *reinterpret_cast<uint4*>(o + 3 * plane) =
        make_uint4(b0.x, b0.y, b1.x, b1.y);
  }
}

extern "C" void qsa_retention_rotate_launch(
    const bf16_t* x, long long xstride, const float* cos_t,
    const float* sin_t, const int* positions, bf16_t* planes, long long rows,
    int H, int D, int DP, int rot, float kscale, int table_len,
    hipStream_t st) {
  // x rows are 16 B aligned and H*D % 4 == 0 on this path
  const bool fast = rot % 16 == 0 && D % 8 == 0;
  int threads = (H * (DP / 8) + 63) / 64 * 64;
  threads = threads > 256 ? 256 : threads;
#define QSA_RR(F)                                                          \
  hipLaunchKernelGGL((qsa_retention_rotate<F>), dim3((unsigned)rows),      \
                     dim3(threads), 0, st, x, xstride, cos_t, sin_t,       \
                     positions, planes, rows, H, D, DP, rot, kscale,       \
                     table_len)
  if (fast) QSA_RR(true); else QSA_RR(false);
#undef QSA_RR
}

// ---------------------------------------------------------------------------
// Step 2: state walk.  Block = (portion, head, 64 value columns); a wave owns
// 16 of the columns and 1/DH of the state rows in accumulators.
//   S_(c+1) = decay^n S_c + sum_j k_j (decay^(n-1-j) v_j)^T
// The state before a chunk is left in the operand order of step 3: for value
// tile vt and 32 dims ks, 16 B per lane (column vt*16 + lane%16; dims
// ks*32 + hi*4 .. +3 and ks*32 + 16 + hi*4 .. +3), so both sides move whole
// 1 KiB lines:  prefix[chunk][head][plane][vt][ks][lane][8]
// ---------------------------------------------------------------------------
template <int KS, int DH>  // DP = 32 * KS, 4 * DH waves
__global__ void __launch_bounds__(256 * DH)
qsa_retention_state(const bf16_t* __restrict__ x, long long xstride,
                    long long voff, const bf16_t* __restrict__ planes,
                    long long rows, const float* __restrict__ log2_decay,
                    float* __restrict__ state, const int* __restrict__ slots,
                    const int* __restrict__ off, const int* __restrict__ start,
                    const int* __restrict__ len,
                    const int* __restrict__ chunk0,
                    u32x4_v* __restrict__ prefix, int H, int D, int E,
                    int EP) {
  constexpr int DP = 32 * KS;
  constexpr int KP = DP + 16;       // LDS pitches (elements)
  constexpr int VP = 64 + 16;
  constexpr int NTH = 256 * DH;
  constexpr int KLD = RC * DP / 8 * 2 / NTH;  // 16 B groups of k per thread
  constexpr int VLD = RC * 8 / NTH;           // ... and of v
  constexpr int NT_ = 2 * KS / DH;            // 16-row tiles per wave
  __shared__ __attribute__((aligned(16))) bf16_t kt[2][RC * KP];
  __shared__ __attribute__((aligned(16))) bf16_t vt[2][RC * VP];
  const int VT = (EP + 63) / 64;
  const int vtile = blockIdx.x % VT;
  const int h = (blockIdx.x / VT) % H;
  const int it = blockIdx.x / (VT * H);
  const int tid = threadIdx.x, lane = tid & 63, wave = (tid >> 6) & 3;
  const int tile0 = (tid >> 8) * NT_;          // this wave's first row tile
  const int col = lane & 15, hi = lane >> 4;
  const int n = len[it], p0 = start[it], r0 = off[it], slot = slots[it];
  const float l2d = log2_decay[h];
  const int v0 = vtile * 64;
  const int e = v0 + wave * 16 + col;          // this lane's value column
  float* S = state + ((long long)slot * H + h) * D * E;
  const long long plane = rows * H * DP;
  const bf16_t* kpl = planes + 2 * plane;

  f32x4_v acc[NT_];
#pragma unroll
  for (int t = 0; t < NT_; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = (tile0 + t) * 16 + hi * 4 + r;
      acc[t][r] = (p0 > 0 && d < D && e < E) ? S[(long long)d * E + e] : 0.f;
    }

  u32x4_v kreg[KLD], vreg[VLD];
#define QSA_FETCH(t0_)                                                        \
  {                                                                           \
    _Pragma("unroll") for (int u = 0; u < KLD; ++u) {                         \
      const int g = tid + u * NTH; /* plane, row, group */                    \
      const int tr = min((t0_) + g / (DP / 8) % RC, n - 1);                   \
      kreg[u] = *reinterpret_cast<const u32x4_v*>(                            \
          kpl + (g / (RC * DP / 8)) * plane +                                 \
          ((long long)(r0 + tr) * H + h) * DP + (g % (DP / 8)) * 8);          \
    }                                                                         \
    _Pragma("unroll") for (int u = 0; u < VLD; ++u) {                         \
      const int g = tid + u * NTH;                                            \
      const int tr = min((t0_) + (g >> 3), n - 1);                            \
      const int cc = min(v0 + (g & 7) * 8, E - 8); /* E % 8 == 0 */           \
      vreg[u] = *reinterpret_cast<const u32x4_v*>(                            \
          x + (long long)(r0 + tr) * xstride + voff + (long long)h * E + cc); \
    }                                                                         \
  }
  QSA_FETCH(0)
  const int nc = (n + RC - 1) / RC;
  for (int c = 0; c < nc; ++c) {
    const int t0 = c * RC;
    const int m = min(RC, n - t0);
    lds_barrier();                   // previous chunk's LDS readers are done
#pragma unroll
    for (int u = 0; u < KLD; ++u) {
      const int g = tid + u * NTH;
      *reinterpret_cast<u32x4_v*>(
          &kt[g / (RC * DP / 8)][g / (DP / 8) % RC * KP +
                                 (g % (DP / 8)) * 8]) = kreg[u];
    }
#pragma unroll
    for (int u = 0; u < VLD; ++u) {
      const int g = tid + u * NTH;
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
    lds_barrier();
    if (c + 1 < nc) QSA_FETCH(t0 + RC)

    // state before this chunk (nothing precedes the first token)
    if ((c > 0 || p0 > 0) && v0 + wave * 16 < EP) {
      const int NT = EP / 16, vt16 = v0 / 16 + wave;
      u32x4_v* ph = prefix +
          ((((long long)(chunk0[it] + c) * H + h) * 2) * NT + vt16) * KS * 64 +
          lane;
      u32x4_v* pl = ph + (long long)NT * KS * 64;
#pragma unroll
      for (int s = 0; s < NT_ / 2; ++s) {
        uint2 a0, b0, a1, b1;
        split4_bf16(acc[2 * s][0], acc[2 * s][1], acc[2 * s][2],
                    acc[2 * s][3], a0, b0);
        split4_bf16(acc[2 * s + 1][0], acc[2 * s + 1][1], acc[2 * s + 1][2],
                    acc[2 * s + 1][3], a1, b1);
        ph[(tile0 / 2 + s) * 64] = (u32x4_v){a0.x, a0.y, a1.x, a1.y};
        pl[(tile0 / 2 + s) * 64] = (u32x4_v){b0.x, b0.y, b1.x, b1.y};
      }
    }
    const float dn = exp2f((float)m * l2d);
#pragma unroll
    for (int t = 0; t < NT_; ++t) acc[t] *= dn;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const bf16x8_v bh =
          lds_frag_tr(vt[0], VP, s * 32, s * 32 + 16, wave * 16, lane);
      const bf16x8_v bl =
          lds_frag_tr(vt[1], VP, s * 32, s * 32 + 16, wave * 16, lane);
#pragma unroll
      for (int t = 0; t < NT_; ++t) {
        const int d0 = (tile0 + t) * 16;
        const bf16x8_v ah =
            lds_frag_tr(kt[0], KP, s * 32, s * 32 + 16, d0, lane);
        const bf16x8_v al =
            lds_frag_tr(kt[1], KP, s * 32, s * 32 + 16, d0, lane);
        acc[t] = mfma_bf16(ah, bh, acc[t]);
        acc[t] = mfma_bf16(ah, bl, acc[t]);
        acc[t] = mfma_bf16(al, bh, acc[t]);
      }
    }
  }
#pragma unroll
  for (int t = 0; t < NT_; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = (tile0 + t) * 16 + hi * 4 + r;
      if (d < D && e < E) S[(long long)d * E + e] = acc[t][r];
    }
}

#undef QSA_FETCH

extern "C" void qsa_retention_state_launch(
    const bf16_t* x, long long xstride, long long voff, const bf16_t* planes,
    long long rows, const float* log2_decay, float* state, const int* slots,
    const int* off, const int* start, const int* len, const int* chunk0,
    void* prefix, int n_items, int H, int D, int DP, int E, int EP,
    hipStream_t st) {
  dim3 grid((unsigned)(n_items * H * ((EP + 63) / 64)));
#define QSA_ST(K, DH)                                                       \
  case K:                                                                   \
    hipLaunchKernelGGL((qsa_retention_state<K, DH>), grid, dim3(256 * DH),  \
                       0, st, x, xstride, voff, planes, rows, log2_decay, state,      \
                       slots, off, start, len, chunk0, (u32x4_v*)prefix, H, \
                       D, E, EP);                                           \
    break;
  switch (DP / 32) { QSA_ST(1, 1) QSA_ST(2, 2) QSA_ST(4, 2) QSA_ST(8, 2) }
#undef QSA_ST
}

// ---------------------------------------------------------------------------
// Step 3: outputs of one (chunk, head) of 64 tokens, O^T in accumulators
// (row = value, column = token):
//   O^T  = decay^(i+1) * (S^T q_i)  +  V^T P^T,   P_ij = q_i.k_j decay^(i-j)
// Wave w of 8 owns the value tiles w, w+8, ... for all 64 tokens, so the state
// before the chunk and V are read once per block.  For P, a wave computes 16
// tokens against 32 keys; P^T leaves that product in
// exactly the operand layout of the next one (the order of the summed index
// is free) and passes through LDS, over the queries that are used up.
// ---------------------------------------------------------------------------
template <int KS, int ET>  // DP = 32*KS, up to 16*ET value columns
__global__ void __launch_bounds__(512)
qsa_retention_out(const bf16_t* __restrict__ x, long long xstride,
                  long long voff, const bf16_t* __restrict__ planes,
                  long long rows, const float* __restrict__ log2_decay,
                  const int* __restrict__ off, const int* __restrict__ start,
                  const int* __restrict__ len,
                  const int* __restrict__ chunk_item,
                  const int* __restrict__ chunk_t0,
                  const u32x4_v* __restrict__ prefix,
                  bf16_t* __restrict__ out, int H, int E, int EP, float eps) {
  constexpr int DP = 32 * KS;
  constexpr int QP = DP + 8;
  constexpr int VP = 16 * ET + 16;
  constexpr int NV = ET <= 8 ? 1 : ET / 8;
  constexpr int QSZ = 2 * RC * QP, PSZ = 2 * 2 * 4 * 64 * 8;
  __shared__ __attribute__((aligned(16))) bf16_t qt[QSZ > PSZ ? QSZ : PSZ];
  __shared__ __attribute__((aligned(16))) bf16_t vt[RC * VP];
  __shared__ float red[8][RC];
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
  const int NT = EP / 16;

#pragma unroll
  for (int u = 0; u < KS; ++u) {
    const int g = tid + u * 512;                    // plane, row, group
    const int p = g / (RC * DP / 8);
    const int row = g / (DP / 8) % RC, c = (g % (DP / 8)) * 8;
    *reinterpret_cast<u32x4_v*>(&qt[(p * RC + row) * QP + c]) =
        *reinterpret_cast<const u32x4_v*>(
            planes + p * plane + ((r0 + min(row, m - 1)) * H + h) * DP + c);
  }
#pragma unroll
  for (int u = 0; u < ET / 4; ++u) {
    const int g = tid + u * 512;
    const int row = g / (2 * ET), c = (g % (2 * ET)) * 8;
    const bool ok = row < m && c < E;               // E % 8 == 0
    const u32x4_v v = *reinterpret_cast<const u32x4_v*>(
        x + (r0 + min(row, m - 1)) * xstride + voff + (long long)h * E +
        (c < E ? c : 0));
    *reinterpret_cast<u32x4_v*>(&vt[row * VP + c]) =
        ok ? v : (u32x4_v){0, 0, 0, 0};
  }
  f32x4_v acc[NV][4];
#pragma unroll
  for (int u = 0; u < NV; ++u)
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) acc[u][rt] = (f32x4_v){0.f, 0.f, 0.f, 0.f};
  lds_barrier();

  if (has_prefix) {                                 // uniform
    const u32x4_v* ph =
        prefix + (((long long)ch * H + h) * 2) * NT * KS * 64 + lane;
    const u32x4_v* pl = ph + (long long)NT * KS * 64;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      bf16x8_v ah[NV], al[NV];
#pragma unroll
      for (int u = 0; u < NV; ++u) {
        const int v = min(wave + 8 * u, NT - 1);    // spare tiles: not stored
        ah[u] = __builtin_bit_cast(bf16x8_v, ph[(v * KS + s) * 64]);
        al[u] = __builtin_bit_cast(bf16x8_v, pl[(v * KS + s) * 64]);
      }
#pragma unroll
      for (int rt = 0; rt < 4; ++rt) {
        const bf16_t* qr = &qt[(rt * 16 + col) * QP + s * 32 + hi * 4];
        const bf16x8_v bh = __builtin_shufflevector(
            *reinterpret_cast<const bf16x4_v*>(qr),
            *reinterpret_cast<const bf16x4_v*>(qr + 16), 0, 1, 2, 3, 4, 5, 6,
            7);
        const bf16x8_v bl = __builtin_shufflevector(
            *reinterpret_cast<const bf16x4_v*>(qr + RC * QP),
            *reinterpret_cast<const bf16x4_v*>(qr + RC * QP + 16), 0, 1, 2, 3,
            4, 5, 6, 7);
#pragma unroll
        for (int u = 0; u < NV; ++u) {
          acc[u][rt] = mfma_bf16(ah[u], bh, acc[u][rt]);
          acc[u][rt] = mfma_bf16(ah[u], bl, acc[u][rt]);
          acc[u][rt] = mfma_bf16(al[u], bh, acc[u][rt]);
        }
      }
    }
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) {
      const float f = exp2f((float)(rt * 16 + col + 1) * l2d);
#pragma unroll
      for (int u = 0; u < NV; ++u) acc[u][rt] *= f;
    }
  }

  // P^T of token tile prt against key tiles 2*ps and 2*ps + 1, keys straight
  // from the planes
  const int prt = wave & 3, ps = wave >> 2;
  const int i = prt * 16 + col;
  u32x4_v pbh, pbl;
  {
    bf16x8_v qh[KS], ql[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const bf16_t* qr = &qt[i * QP + s * 32 + hi * 8];
      qh[s] = *reinterpret_cast<const bf16x8_v*>(qr);
      ql[s] = *reinterpret_cast<const bf16x8_v*>(qr + RC * QP);
    }
    uint2 ph[2], pl[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int pt = ps * 2 + u;
      f32x4_v sc = {0.f, 0.f, 0.f, 0.f};
      if (pt <= prt) {                              // uniform over the wave
        const bf16_t* kr = planes + 2 * plane +
            ((r0 + min(pt * 16 + col, m - 1)) * H + h) * DP + hi * 8;
#pragma unroll
        for (int s = 0; s < KS; ++s) {
          const bf16x8_v ah = *reinterpret_cast<const bf16x8_v*>(kr + s * 32);
          const bf16x8_v al =
              *reinterpret_cast<const bf16x8_v*>(kr + plane + s * 32);
          sc = mfma_bf16(ah, qh[s], sc);
          sc = mfma_bf16(ah, ql[s], sc);
          sc = mfma_bf16(al, qh[s], sc);
        }
      }
      float w[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = pt * 16 + hi * 4 + r;
        const bool ok = j <= i && j < m;
        w[r] = ok ? sc[r] * exp2f((float)(i - j) * l2d) : 0.f;
      }
      split4_bf16(w[0], w[1], w[2], w[3], ph[u], pl[u]);
    }
    pbh = (u32x4_v){ph[0].x, ph[0].y, ph[1].x, ph[1].y};
    pbl = (u32x4_v){pl[0].x, pl[0].y, pl[1].x, pl[1].y};
  }
  lds_barrier();                                    // all queries are read
  u32x4_v* pt = reinterpret_cast<u32x4_v*>(qt);     // [plane][s2][rt][lane]
  pt[wave * 64 + lane] = pbh;
  pt[(8 + wave) * 64 + lane] = pbl;
  lds_barrier();
#pragma unroll
  for (int s2 = 0; s2 < 2; ++s2)
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int v = min(wave + 8 * u, NT - 1);
      const bf16x8_v av = lds_frag_tr(vt, VP, s2 * 32, s2 * 32 + 16, v * 16,
                                      lane);
#pragma unroll
      for (int rt = 2 * s2; rt < 4; ++rt) {
        const bf16x8_v bh = __builtin_bit_cast(
            bf16x8_v, pt[(s2 * 4 + rt) * 64 + lane]);
        const bf16x8_v bl = __builtin_bit_cast(
            bf16x8_v, pt[(8 + s2 * 4 + rt) * 64 + lane]);
        acc[u][rt] = mfma_bf16(av, bh, acc[u][rt]);
        acc[u][rt] = mfma_bf16(av, bl, acc[u][rt]);
      }
    }

  // per-token rms over the value columns, gate, store
#pragma unroll
  for (int rt = 0; rt < 4; ++rt) {
    float ss = 0.f;
#pragma unroll
    for (int u = 0; u < NV; ++u)
      if (wave + 8 * u < NT) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          ss = fmaf(acc[u][rt][r], acc[u][rt][r], ss);
      }
    ss += __shfl_xor(ss, 16, QSA_WAVE);
    ss += __shfl_xor(ss, 32, QSA_WAVE);
    if (hi == 0) red[wave][rt * 16 + col] = ss;
  }
  lds_barrier();
#pragma unroll
  for (int rt = 0; rt < 4; ++rt) {
    const int t = rt * 16 + col;
    const float ss = ((red[0][t] + red[1][t]) + (red[2][t] + red[3][t])) +
                     ((red[4][t] + red[5][t]) + (red[6][t] + red[7][t]));
    const float inv = 1.f / sqrtf(ss / (float)E + eps);
    if (t < m) {
      const bf16_t* g = x + (r0 + t) * xstride + voff + (long long)H * E +
                        (long long)h * E;
      bf16_t* orow = out + ((r0 + t) * H + h) * E;
#pragma unroll
      for (int u = 0; u < NV; ++u) {
        const int e0 = (wave + 8 * u) * 16 + hi * 4;
        if (e0 < E) {                               // E % 8 == 0
          float gv[4], o[4];
          ldv<bf16_t, 4>(g + e0, gv);
#pragma unroll
          for (int r = 0; r < 4; ++r)
            o[r] = acc[u][rt][r] * inv * (gv[r] / (1.f + __expf(-gv[r])));
          stv<bf16_t, 4>(orow + e0, o);
        }
      }
    }
  }
}

extern "C" void qsa_retention_out_launch(
    const bf16_t* x, long long xstride, long long voff, const bf16_t* planes,
    long long rows, const float* log2_decay, const int* off,
    const int* start, const int* len, const int* chunk_item,
    const int* chunk_t0, const void* prefix, long long n_chunks,
    bf16_t* out, int H, int DP, int E, int EP, float eps, hipStream_t st) {
  dim3 grid((unsigned)(n_chunks * H));
#define QSA_RO(K, V)                                                        \
  hipLaunchKernelGGL((qsa_retention_out<K, V>), grid, dim3(512), 0, st, x,  \
                     xstride, voff, planes, rows, log2_decay, off, start,   \
                     len, chunk_item, chunk_t0, (const u32x4_v*)prefix,     \
                     out, H, E, EP, eps)
#define QSA_RO_E(K)                                                         \
  if (EP <= 64) QSA_RO(K, 4);                                               \
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
