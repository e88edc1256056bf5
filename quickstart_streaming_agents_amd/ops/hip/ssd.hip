// State-space duality (a scalar, input-dependent decay per head) for gfx950.
//
//   dt_t = softplus(raw_t + dt_bias)                        per head
//   S_t  = exp(-A dt_t) S_(t-1) + dt_t B_t x_t^T            S [N, P], f32
//   y_t  = S_t^T C_t + D x_t,   out = y * silu(z)
//
// x [H*P], B [G*N], C [G*N] of a token are one dense row of the convolution's
// output; head h reads B and C of group h / (H / G).  z and raw dt are columns
// of the projection row.  State: [slots, H, N, P] f32, one slot per live
// sequence, taken as zero at position 0 (slots need no clearing).
//
// Kernels
//   qsa_ssd_decode   one token per row: step size, decay, update, read-out and
//                    gate in one pass over the state (HBM-bound).
//   qsa_ssd_seq      token loop per (portion, head), any size and storage
//                    type; the f32 path.
//   chunked prefill (bf16 storage, matrix cores), chunks of 64 tokens; with
//   c_i the running sum of the log decay inside a chunk (in powers of two):
//     qsa_ssd_steps  dt and c of every token
//     qsa_ssd_state  walks the chunks of a portion, state tile in
//                    accumulators; leaves the state before each chunk as
//                    hi/lo matrix-core operands
//     qsa_ssd_out    per (chunk, head):
//                    2^c_i S^T C_i + sum_j<=i (C_i.B_j) 2^(c_i-c_j) dt_j x_j
//   B, C and x are bf16 already; what is rounded on the way to the matrix
//   cores (decayed x, state, intra-chunk weights) is a bf16 hi/lo pair, so the
//   chunked result agrees with the token loop to about 2^-16.
//   qsa_part_norm    rms norm in equal parts of a row, with a weight
#include "lm_common.h"

#define RC 64  // tokens per chunk
#define LOG2E 1.4426950408889634f

__device__ __forceinline__ float softplus_f(float v) {
  return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v)));
}

// ---------------------------------------------------------------------------
// Decode: one block per (row, head).
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__global__ void __launch_bounds__(1024)
qsa_ssd_decode(const T* __restrict__ u, long long ustride, int zoff,
               int dtoff, const T* __restrict__ xbc,
               const float* __restrict__ A, const float* __restrict__ dt_bias,
               const float* __restrict__ Dskip, float* __restrict__ state,
               const int* __restrict__ slots,
               const int* __restrict__ seq_lens, T* __restrict__ out, int H,
               int N, int P, int G, int CW) {
  extern __shared__ float sm[];
  float* bs = sm;                 // N
  float* cs = bs + N;             // N
  float* red = cs + (2 * N + 3) / 4 * 4 - N;  // threads * VEC
  const int b = blockIdx.x / H, h = blockIdx.x % H;
  const int tid = threadIdx.x, nth = blockDim.x;
  const int pos = seq_lens[b] - 1;
  const int slot = slots[b];
  T* orow = out + ((long long)b * H + h) * P;
  if (pos < 0 || slot < 0) {                       // uniform over the block
    for (int e = tid; e < P; e += nth) stf<T>(orow + e, 0.f);
    return;
  }
  const int g = h / (H / G);
  const T* ur = u + (long long)b * ustride;
  const T* xr = xbc + (long long)b * (H * P + 2 * G * N);
  const T* x = xr + (long long)h * P;
  const T* z = ur + zoff + (long long)h * P;
  const T* Bp = xr + (long long)H * P + (long long)g * N;
  const T* Cp = Bp + (long long)G * N;
  const float dt = softplus_f(ldf<T>(ur + dtoff + h) + dt_bias[h]);
  const float dec = expf(-A[h] * dt);
  for (int d = tid; d < N; d += nth) {
    bs[d] = ldf<T>(Bp + d) * dt;
    cs[d] = ldf<T>(Cp + d);
  }
  __syncthreads();
  const bool fresh = pos == 0;
  float* S = state + ((long long)slot * H + h) * N * P;
  const int GR = nth / CW;         // row groups
  const int c0 = tid % CW, g0 = tid / CW;
  const int NV = P / VEC;
  const float dk = Dskip[h];
  for (int cb = 0; cb < NV; cb += CW) {
    const int c = cb + c0;
    float acc[VEC], xv[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) acc[j] = 0.f;
    if (c < NV) {
      ldv<T, VEC>(x + c * VEC, xv);
      float* sp = S + c * VEC;
#pragma unroll 4
      for (int d = g0; d < N; d += GR) {
        float s[VEC];
        if (fresh) {
#pragma unroll
          for (int j = 0; j < VEC; ++j) s[j] = 0.f;
        } else {
          ldv<float, VEC>(sp + (long long)d * P, s);
        }
        const float kd = bs[d], qd = cs[d];
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          s[j] = fmaf(dec, s[j], kd * xv[j]);
          acc[j] = fmaf(qd, s[j], acc[j]);
        }
        stv<float, VEC>(sp + (long long)d * P, s);
      }
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) red[tid * VEC + j] = acc[j];
    __syncthreads();
    if (g0 == 0 && c < NV) {
      for (int gg = 1; gg < GR; ++gg)
#pragma unroll
        for (int j = 0; j < VEC; ++j) acc[j] += red[(gg * CW + c0) * VEC + j];
      float zv[VEC];
      ldv<T, VEC>(z + c * VEC, zv);
#pragma unroll
      for (int j = 0; j < VEC; ++j)
        acc[j] = (acc[j] + dk * xv[j]) * silu_f(zv[j]);
      stv<T, VEC>(orow + c * VEC, acc);
    }
    __syncthreads();
  }
}

extern "C" void qsa_ssd_decode_launch(
    const void* u, long long ustride, int zoff, int dtoff, const void* xbc,
    const float* A, const float* dt_bias, const float* Dskip, float* state,
    const int* slots, const int* seq_lens, void* out, int B, int H, int N,
    int P, int G, int f32, int vec4, hipStream_t st) {
  const int nv = vec4 ? P / 4 : P;
  int cw = 1;
  while (cw < nv && cw < 256) cw <<= 1;
  // few blocks: wide ones, so that enough of the state is in flight
  const int threads =
      (long long)B * H <= 512 && (long long)N * P >= 16384 ? 1024 : 256;
  const size_t lds = sizeof(float) *
      ((2 * (size_t)N + 3) / 4 * 4 + threads * (vec4 ? 4 : 1));
#define QSA_SD(T, V)                                                         \
  hipLaunchKernelGGL((qsa_ssd_decode<T, V>), dim3((unsigned)(B * H)),        \
                     dim3(threads), lds, st, (const T*)u, ustride, zoff,     \
                     dtoff, (const T*)xbc, A, dt_bias, Dskip, state, slots,  \
                     seq_lens, (T*)out, H, N, P, G, cw)
  if (f32) { if (vec4) QSA_SD(float, 4); else QSA_SD(float, 1); }
  else     { if (vec4) QSA_SD(bf16_t, 4); else QSA_SD(bf16_t, 1); }
#undef QSA_SD
}

// ---------------------------------------------------------------------------
// Token loop over a portion: one block per (portion, head).  CW threads cover
// the columns, the others split the state's rows; the tile stays in LDS when
// it fits.
// ---------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256)
qsa_ssd_seq(const T* __restrict__ u, long long ustride, int zoff, int dtoff,
            const T* __restrict__ xbc, const float* __restrict__ A,
            const float* __restrict__ dt_bias,
            const float* __restrict__ Dskip, float* __restrict__ state,
            const int* __restrict__ slots, const int* __restrict__ off,
            const int* __restrict__ start, const int* __restrict__ len,
            T* __restrict__ out, int H, int N, int P, int G, int CW,
            int in_lds) {
  extern __shared__ float sm[];
  float* bs = sm;                 // N
  float* cs = bs + N;             // N
  float* red = cs + N;            // 256
  float* tile = red + 256;
  const int it = blockIdx.x / H, h = blockIdx.x % H;
  const int tid = threadIdx.x;
  const int n = len[it], p0 = start[it], r0 = off[it], slot = slots[it];
  if (slot < 0) return;
  const int g = h / (H / G);
  const int CX = H * P + 2 * G * N;
  float* Sg = state + ((long long)slot * H + h) * N * P;
  float* S = in_lds ? tile : Sg;
  for (int i = tid; i < N * P; i += 256)
    if (p0 == 0) S[i] = 0.f;
    else if (in_lds) S[i] = Sg[i];
  const int GR = 256 / CW, c0 = tid % CW, g0 = tid / CW;
  const float ah = A[h], bh = dt_bias[h], dk = Dskip[h];
  for (int t = 0; t < n; ++t) {
    const T* ur = u + (long long)(r0 + t) * ustride;
    const T* xr = xbc + (long long)(r0 + t) * CX;
    const T* x = xr + (long long)h * P;
    const T* Bp = xr + (long long)H * P + (long long)g * N;
    const float dt = softplus_f(ldf<T>(ur + dtoff + h) + bh);
    const float dec = expf(-ah * dt);
    __syncthreads();   // previous token's readers are done
    for (int d = tid; d < N; d += 256) {
      bs[d] = ldf<T>(Bp + d) * dt;
      cs[d] = ldf<T>(Bp + (long long)G * N + d);
    }
    __syncthreads();
    for (int cb = 0; cb < P; cb += CW) {
      const int e = cb + c0;
      float acc = 0.f, xe = 0.f;
      if (e < P) {
        xe = ldf<T>(x + e);
        for (int d = g0; d < N; d += GR) {
          const float s = fmaf(dec, S[d * P + e], bs[d] * xe);
          S[d * P + e] = s;
          acc = fmaf(cs[d], s, acc);
        }
      }
      if (GR > 1) {                                // uniform
        red[tid] = acc;
        __syncthreads();
        if (g0 == 0)
          for (int gg = 1; gg < GR; ++gg) acc += red[gg * CW + c0];
        __syncthreads();
      }
      if (g0 == 0 && e < P)
        stf<T>(out + ((long long)(r0 + t) * H + h) * P + e,
               (acc + dk * xe) *
                   silu_f(ldf<T>(ur + zoff + (long long)h * P + e)));
    }
  }
  if (in_lds) {
    __syncthreads();
    for (int i = tid; i < N * P; i += 256) Sg[i] = S[i];
  }
}

extern "C" void qsa_ssd_seq_launch(
    const void* u, long long ustride, int zoff, int dtoff, const void* xbc,
    const float* A, const float* dt_bias, const float* Dskip, float* state,
    const int* slots, const int* off, const int* start, const int* len,
    void* out, int n_items, int H, int N, int P, int G, int f32,
    hipStream_t st) {
  size_t lds = sizeof(float) * (2 * (size_t)N + 256);
  const size_t with_tile = lds + sizeof(float) * (size_t)N * P;
  const int in_lds = with_tile <= 60 * 1024;
  if (in_lds) lds = with_tile;
  int cw = 1;
  while (cw < P && cw < 256) cw <<= 1;
#define QSA_SS(T)                                                           \
  hipLaunchKernelGGL((qsa_ssd_seq<T>), dim3((unsigned)(n_items * H)),       \
                     dim3(256), lds, st, (const T*)u, ustride, zoff, dtoff, \
                     (const T*)xbc, A, dt_bias, Dskip, state, slots, off,   \
                     start, len, (T*)out, H, N, P, G, cw, in_lds)
  if (f32) QSA_SS(float); else QSA_SS(bf16_t);
#undef QSA_SS
}

// ---------------------------------------------------------------------------
// Chunked prefill, step 1: per (chunk, head) 64 step sizes and the running
// sums of the log2 decay; places past the portion's end have dt = 0.
// steps[chunk][head][2][64]
// ---------------------------------------------------------------------------
__global__ void __launch_bounds__(256)
qsa_ssd_steps(const bf16_t* __restrict__ u, long long ustride, int dtoff,
              const float* __restrict__ A, const float* __restrict__ dt_bias,
              const int* __restrict__ off, const int* __restrict__ len,
              const int* __restrict__ chunk_item,
              const int* __restrict__ chunk_t0, float* __restrict__ steps,
              int H) {
  const int ch = blockIdx.x;
  const int it = chunk_item[ch], t0 = chunk_t0[ch];
  const int m = min(RC, len[it] - t0);
  const int lane = threadIdx.x & 63;
  const bf16_t* row = u +
      (long long)(off[it] + t0 + min(lane, m - 1)) * ustride + dtoff;
  for (int h = threadIdx.x >> 6; h < H; h += 4) {
    float dt = softplus_f(ldf<bf16_t>(row + h) + dt_bias[h]);
    dt = lane < m ? dt : 0.f;
    float c = -A[h] * dt * LOG2E;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float v = __shfl_up(c, o, QSA_WAVE);
      if (lane >= o) c += v;
    }
    float* s = steps + ((long long)ch * H + h) * 2 * RC + lane;
    s[0] = dt;
    s[RC] = c;
  }
}

extern "C" void qsa_ssd_steps_launch(const bf16_t* u, long long ustride,
                                     int dtoff, const float* A,
                                     const float* dt_bias, const int* off,
                                     const int* len, const int* chunk_item,
                                     const int* chunk_t0, float* steps,
                                     int n_chunks, int H, hipStream_t st) {
  hipLaunchKernelGGL(qsa_ssd_steps, dim3((unsigned)n_chunks), dim3(256), 0,
                     st, u, ustride, dtoff, A, dt_bias, off, len, chunk_item,
                     chunk_t0, steps, H);
}

// ---------------------------------------------------------------------------
// Step 2: state walk.  Block = (portion, head, 64 value columns); a wave owns
// 16 of the columns and 1/DH of the state rows in accumulators.
//   S' = 2^c_last S + sum_j B_j (2^(c_last - c_j) dt_j x_j)^T
// The state before a chunk is left in the operand order of step 3: for value
// tile vt and 32 rows ks, 16 B per lane (column vt*16 + lane%16; rows
// ks*32 + hi*4 .. +3 and ks*32 + 16 + hi*4 .. +3), so both sides move whole
// 1 KiB lines:  prefix[chunk][head][plane][vt][ks][lane][8]
// ---------------------------------------------------------------------------
template <int KS, int DH>  // DP = 32 * KS >= N, 4 * DH waves
__global__ void __launch_bounds__(256 * DH)
qsa_ssd_state(const bf16_t* __restrict__ xbc, const float* __restrict__ steps,
              float* __restrict__ state, const int* __restrict__ slots,
              const int* __restrict__ off, const int* __restrict__ start,
              const int* __restrict__ len, const int* __restrict__ chunk0,
              u32x4_v* __restrict__ prefix, int H, int N, int P, int G,
              int EP) {
  constexpr int DP = 32 * KS;
  constexpr int KP = DP + 16;       // LDS pitches (elements)
  constexpr int VP = 64 + 16;
  constexpr int NTH = 256 * DH;
  constexpr int KLD = RC * DP / 8 / NTH;      // 16 B groups of B per thread
  constexpr int VLD = RC * 8 / NTH;           // ... and of x
  constexpr int NT_ = 2 * KS / DH;            // 16-row tiles per wave
  __shared__ __attribute__((aligned(16))) bf16_t kt[RC * KP];
  __shared__ __attribute__((aligned(16))) bf16_t vt[2][RC * VP];
  const int VT = (EP + 63) / 64;
  const int vtile = blockIdx.x % VT;
  const int h = (blockIdx.x / VT) % H;
  const int it = blockIdx.x / (VT * H);
  const int tid = threadIdx.x, lane = tid & 63, wave = (tid >> 6) & 3;
  const int tile0 = (tid >> 8) * NT_;          // this wave's first row tile
  const int col = lane & 15, hi = lane >> 4;
  const int n = len[it], p0 = start[it], r0 = off[it], slot = slots[it];
  const int v0 = vtile * 64;
  const int e = v0 + wave * 16 + col;          // this lane's value column
  const int CX = H * P + 2 * G * N;
  float* S = state + ((long long)slot * H + h) * N * P;
  const bf16_t* bp = xbc + H * P + (h / (H / G)) * N;
  const bf16_t* xp = xbc + h * P;

  f32x4_v acc[NT_];
#pragma unroll
  for (int t = 0; t < NT_; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = (tile0 + t) * 16 + hi * 4 + r;
      acc[t][r] = (p0 > 0 && d < N && e < P) ? S[(long long)d * P + e] : 0.f;
    }

  u32x4_v kreg[KLD], vreg[VLD];
  float fdt[VLD], fcum[VLD], flast;
  auto fetch = [&](int c) {
    const int t0 = c * RC;
    const float* sp = steps + ((long long)(chunk0[it] + c) * H + h) * 2 * RC;
    flast = sp[2 * RC - 1];
#pragma unroll
    for (int i = 0; i < KLD; ++i) {
      const int g = tid + i * NTH;
      const int tr = min(t0 + g / (DP / 8), n - 1);
      const int cc = (g % (DP / 8)) * 8;           // N % 8 == 0
      const u32x4_v v = *reinterpret_cast<const u32x4_v*>(
          bp + (long long)(r0 + tr) * CX + (cc < N ? cc : 0));
      kreg[i] = cc < N ? v : (u32x4_v){0, 0, 0, 0};
    }
#pragma unroll
    for (int i = 0; i < VLD; ++i) {
      const int g = tid + i * NTH;
      const int tr = min(t0 + (g >> 3), n - 1);
      const int cc = min(v0 + (g & 7) * 8, P - 8); // P % 8 == 0
      vreg[i] = *reinterpret_cast<const u32x4_v*>(
          xp + (long long)(r0 + tr) * CX + cc);
      fdt[i] = sp[g >> 3];
      fcum[i] = sp[RC + (g >> 3)];
    }
  };
  fetch(0);
  const int nc = (n + RC - 1) / RC;
  for (int c = 0; c < nc; ++c) {
    lds_barrier();                   // previous chunk's LDS readers are done
#pragma unroll
    for (int i = 0; i < KLD; ++i) {
      const int g = tid + i * NTH;
      *reinterpret_cast<u32x4_v*>(
          &kt[g / (DP / 8) * KP + (g % (DP / 8)) * 8]) = kreg[i];
    }
#pragma unroll
    for (int i = 0; i < VLD; ++i) {
      const int g = tid + i * NTH;
      const int row = g >> 3, cc = (g & 7) * 8;
      // dt is zero past the portion's end
      const float f = v0 + cc < P ? fdt[i] * exp2f(flast - fcum[i]) : 0.f;
      const u32x4_v pk = vreg[i];
      const float2 v01 = bf16x2_to_f32x2(pk.x), v23 = bf16x2_to_f32x2(pk.y);
      const float2 v45 = bf16x2_to_f32x2(pk.z), v67 = bf16x2_to_f32x2(pk.w);
      uint2 h0, l0, h1, l1;
      split4_bf16(v01.x * f, v01.y * f, v23.x * f, v23.y * f, h0, l0);
      split4_bf16(v45.x * f, v45.y * f, v67.x * f, v67.y * f, h1, l1);
      *reinterpret_cast<uint4*>(&vt[0][row * VP + cc]) =
          make_uint4(h0.x, h0.y, h1.x, h1.y);
      *reinterpret_cast<uint4*>(&vt[1][row * VP + cc]) =
          make_uint4(l0.x, l0.y, l1.x, l1.y);
    }
    const float dn = exp2f(flast);
    lds_barrier();
    if (c + 1 < nc) fetch(c + 1);

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
        const bf16x8_v a =
            lds_frag_tr(kt, KP, s * 32, s * 32 + 16, (tile0 + t) * 16, lane);
        acc[t] = mfma_bf16(a, bh, acc[t]);
        acc[t] = mfma_bf16(a, bl, acc[t]);
      }
    }
  }
#pragma unroll
  for (int t = 0; t < NT_; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = (tile0 + t) * 16 + hi * 4 + r;
      if (d < N && e < P) S[(long long)d * P + e] = acc[t][r];
    }
}

extern "C" void qsa_ssd_state_launch(
    const bf16_t* xbc, const float* steps, float* state, const int* slots,
    const int* off, const int* start, const int* len, const int* chunk0,
    void* prefix, int n_items, int H, int N, int DP, int P, int EP, int G,
    hipStream_t st) {
  dim3 grid((unsigned)(n_items * H * ((EP + 63) / 64)));
#define QSA_ST(K, DH)                                                       \
  case K:                                                                   \
    hipLaunchKernelGGL((qsa_ssd_state<K, DH>), grid, dim3(256 * DH), 0, st, \
                       xbc, steps, state, slots, off, start, len, chunk0,   \
                       (u32x4_v*)prefix, H, N, P, G, EP);                   \
    break;
  switch (DP / 32) { QSA_ST(1, 1) QSA_ST(2, 2) QSA_ST(4, 2) QSA_ST(8, 2) }
#undef QSA_ST
}

// ---------------------------------------------------------------------------
// Step 3: outputs of one (chunk, head) of 64 tokens, O^T in accumulators
// (row = value, column = token).  8 waves = VW shares of the value tiles x
// shares of the token tiles.  For the intra-chunk weights, a wave computes 16
// tokens against 32 keys; their transpose leaves that product in exactly the
// operand layout of the next one (the order of the summed index is free) and
// passes through LDS, over the rows of C that are used up.
// ---------------------------------------------------------------------------
template <int KS, int ET>  // N <= 32*KS, P <= 16*ET
__global__ void __launch_bounds__(512)
qsa_ssd_out(const bf16_t* __restrict__ u, long long ustride, int zoff,
            const bf16_t* __restrict__ xbc, const float* __restrict__ steps,
            const float* __restrict__ Dskip, const int* __restrict__ off,
            const int* __restrict__ start, const int* __restrict__ len,
            const int* __restrict__ chunk_item,
            const int* __restrict__ chunk_t0,
            const u32x4_v* __restrict__ prefix, bf16_t* __restrict__ out,
            int H, int N, int P, int G, int EP) {
  constexpr int DP = 32 * KS;
  constexpr int QP = DP + 8;
  constexpr int VP = 16 * ET + 16;
  constexpr int VW = ET < 8 ? ET : 8;
  constexpr int NV = ET / VW;                       // value tiles per wave
  constexpr int TT = 4 * VW / 8;                    // token tiles per wave
  constexpr int CL = (64 * DP / 8 + 511) / 512, XL = (128 * ET + 511) / 512;
  constexpr int QSZ = RC * QP, PSZ = 2 * 2 * 4 * 64 * 8;
  __shared__ __attribute__((aligned(16))) bf16_t qt[QSZ > PSZ ? QSZ : PSZ];
  __shared__ __attribute__((aligned(16))) bf16_t vt[RC * VP];
  __shared__ float sdt[RC], scum[RC];
  const int h = blockIdx.x % H;
  const int ch = blockIdx.x / H;
  const int it = chunk_item[ch], t0 = chunk_t0[ch];
  const int m = min(RC, len[it] - t0);
  const long long r0 = off[it] + t0;
  const bool has_prefix = t0 > 0 || start[it] > 0;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int vw = wave % VW, tw = wave / VW;
  const int col = lane & 15, hi = lane >> 4;
  const int NT = EP / 16;
  const int CX = H * P + 2 * G * N;
  const bf16_t* bp = xbc + H * P + (h / (H / G)) * N;
  const bf16_t* cp = bp + G * N;

  if (tid < 2 * RC) {
    const float v = steps[((long long)ch * H + h) * 2 * RC + tid];
    if (tid < RC) sdt[tid] = v; else scum[tid - RC] = v;
  }
#pragma unroll
  for (int i = 0; i < CL; ++i) {
    const int g = tid + i * 512;
    const int row = g / (DP / 8), c = (g % (DP / 8)) * 8;
    if (row < RC) {
      const u32x4_v v = *reinterpret_cast<const u32x4_v*>(
          cp + (r0 + min(row, m - 1)) * CX + (c < N ? c : 0));
      *reinterpret_cast<u32x4_v*>(&qt[row * QP + c]) =
          c < N ? v : (u32x4_v){0, 0, 0, 0};
    }
  }
#pragma unroll
  for (int i = 0; i < XL; ++i) {
    const int g = tid + i * 512;
    const int row = g / (2 * ET), c = (g % (2 * ET)) * 8;
    const bool ok = row < m && c < P;               // P % 8 == 0
    const u32x4_v v = *reinterpret_cast<const u32x4_v*>(
        xbc + (r0 + min(row, m - 1)) * CX + (long long)h * P +
        (c < P ? c : 0));
    if (row < RC)
      *reinterpret_cast<u32x4_v*>(&vt[row * VP + c]) =
          ok ? v : (u32x4_v){0, 0, 0, 0};
  }
  f32x4_v acc[NV][TT];
#pragma unroll
  for (int v = 0; v < NV; ++v)
#pragma unroll
    for (int t = 0; t < TT; ++t) acc[v][t] = (f32x4_v){0.f, 0.f, 0.f, 0.f};
  lds_barrier();

  if (has_prefix) {                                 // uniform
    const u32x4_v* ph =
        prefix + (((long long)ch * H + h) * 2) * NT * KS * 64 + lane;
    const u32x4_v* pl = ph + (long long)NT * KS * 64;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      bf16x8_v ah[NV], al[NV];
#pragma unroll
      for (int v = 0; v < NV; ++v) {
        const int k = min(vw + VW * v, NT - 1);     // spare tiles: not stored
        ah[v] = __builtin_bit_cast(bf16x8_v, ph[(k * KS + s) * 64]);
        al[v] = __builtin_bit_cast(bf16x8_v, pl[(k * KS + s) * 64]);
      }
#pragma unroll
      for (int t = 0; t < TT; ++t) {
        const bf16_t* qr =
            &qt[((tw * TT + t) * 16 + col) * QP + s * 32 + hi * 4];
        const bf16x8_v b = __builtin_shufflevector(
            *reinterpret_cast<const bf16x4_v*>(qr),
            *reinterpret_cast<const bf16x4_v*>(qr + 16), 0, 1, 2, 3, 4, 5, 6,
            7);
#pragma unroll
        for (int v = 0; v < NV; ++v) {
          acc[v][t] = mfma_bf16(ah[v], b, acc[v][t]);
          acc[v][t] = mfma_bf16(al[v], b, acc[v][t]);
        }
      }
    }
#pragma unroll
    for (int t = 0; t < TT; ++t) {
      const float f = exp2f(scum[(tw * TT + t) * 16 + col]);
#pragma unroll
      for (int v = 0; v < NV; ++v) acc[v][t] *= f;
    }
  }

  // weights^T of token tile prt against key tiles 2*ps and 2*ps + 1, the rows
  // of B straight from memory
  const int prt = wave & 3, ps = wave >> 2;
  const int i = prt * 16 + col;
  u32x4_v pbh, pbl;
  {
    bf16x8_v q[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s)
      q[s] = *reinterpret_cast<const bf16x8_v*>(&qt[i * QP + s * 32 + hi * 8]);
    uint2 ph[2], pl[2];
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      const int pt = ps * 2 + k;
      f32x4_v sc = {0.f, 0.f, 0.f, 0.f};
      if (pt <= prt) {                              // uniform over the wave
        const bf16_t* kr = bp + (r0 + min(pt * 16 + col, m - 1)) * CX;
#pragma unroll
        for (int s = 0; s < KS; ++s) {
          const int d = s * 32 + hi * 8;            // past N: times zero
          const bf16x8_v a =
              *reinterpret_cast<const bf16x8_v*>(kr + (d < N ? d : 0));
          sc = mfma_bf16(a, q[s], sc);
        }
      }
      float w[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = pt * 16 + hi * 4 + r;
        w[r] = j <= i ? sc[r] * exp2f(scum[i] - scum[j]) * sdt[j] : 0.f;
      }
      split4_bf16(w[0], w[1], w[2], w[3], ph[k], pl[k]);
    }
    pbh = (u32x4_v){ph[0].x, ph[0].y, ph[1].x, ph[1].y};
    pbl = (u32x4_v){pl[0].x, pl[0].y, pl[1].x, pl[1].y};
  }
  lds_barrier();                                    // all of C is read
  u32x4_v* pt = reinterpret_cast<u32x4_v*>(qt);     // [plane][s2][rt][lane]
  pt[wave * 64 + lane] = pbh;
  pt[(8 + wave) * 64 + lane] = pbl;
  lds_barrier();
#pragma unroll
  for (int s2 = 0; s2 < 2; ++s2)
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int k = min(vw + VW * v, NT - 1);
      const bf16x8_v av = lds_frag_tr(vt, VP, s2 * 32, s2 * 32 + 16, k * 16,
                                      lane);
#pragma unroll
      for (int t = 0; t < TT; ++t) {
        const int rt = tw * TT + t;
        if (rt < 2 * s2) continue;                  // keys after the tokens
        const bf16x8_v bh = __builtin_bit_cast(
            bf16x8_v, pt[(s2 * 4 + rt) * 64 + lane]);
        const bf16x8_v bl = __builtin_bit_cast(
            bf16x8_v, pt[(8 + s2 * 4 + rt) * 64 + lane]);
        acc[v][t] = mfma_bf16(av, bh, acc[v][t]);
        acc[v][t] = mfma_bf16(av, bl, acc[v][t]);
      }
    }

  // skip, gate, store
  const float dk = Dskip[h];
#pragma unroll
  for (int t = 0; t < TT; ++t) {
    const int tok = (tw * TT + t) * 16 + col;
    if (tok < m) {
      const bf16_t* z = u + (r0 + tok) * ustride + zoff + (long long)h * P;
      bf16_t* orow = out + ((r0 + tok) * H + h) * P;
#pragma unroll
      for (int v = 0; v < NV; ++v) {
        const int e0 = (vw + VW * v) * 16 + hi * 4;
        if (e0 < P) {
          float zv[4], xv[4], o[4];
          ldv<bf16_t, 4>(z + e0, zv);
          ldv<bf16_t, 4>(&vt[tok * VP + e0], xv);
#pragma unroll
          for (int r = 0; r < 4; ++r)
            o[r] = (acc[v][t][r] + dk * xv[r]) *
                   (zv[r] / (1.f + __expf(-zv[r])));
          stv<bf16_t, 4>(orow + e0, o);
        }
      }
    }
  }
}

extern "C" void qsa_ssd_out_launch(
    const bf16_t* u, long long ustride, int zoff, const bf16_t* xbc,
    const float* steps, const float* Dskip, const int* off, const int* start,
    const int* len, const int* chunk_item, const int* chunk_t0,
    const void* prefix, int n_chunks, bf16_t* out, int H, int N, int DP,
    int P, int EP, int G, hipStream_t st) {
  dim3 grid((unsigned)((long long)n_chunks * H));
#define QSA_SO(K, V)                                                        \
  hipLaunchKernelGGL((qsa_ssd_out<K, V>), grid, dim3(512), 0, st, u,        \
                     ustride, zoff, xbc, steps, Dskip, off, start, len,     \
                     chunk_item, chunk_t0, (const u32x4_v*)prefix, out, H,  \
                     N, P, G, EP)
#define QSA_SO_E(K)                                                         \
  if (EP <= 32) QSA_SO(K, 2);                                               \
  else if (EP <= 64) QSA_SO(K, 4);                                          \
  else if (EP <= 128) QSA_SO(K, 8);                                         \
  else QSA_SO(K, 16)
  switch (DP / 32) {
    case 1: QSA_SO_E(1); break;
    case 2: QSA_SO_E(2); break;
    case 4: QSA_SO_E(4); break;
    case 8: QSA_SO_E(8); break;
  }
#undef QSA_SO_E
#undef QSA_SO
}

// ---------------------------------------------------------------------------
// RMS norm of a row in equal parts, times w (f32).  A wave per part for short
// ones, a block otherwise.
// ---------------------------------------------------------------------------
template <typename T, int VEC, bool WAVE>
__global__ void __launch_bounds__(256)
qsa_part_norm(const T* __restrict__ x, const float* __restrict__ w,
              T* __restrict__ out, long long ostride, long long units,
              int parts, int n, float eps) {
  __shared__ float scratch[8];
  const int tid = WAVE ? threadIdx.x & 63 : threadIdx.x;
  const int nth = WAVE ? 64 : blockDim.x;
  const long long unit =
      WAVE ? (long long)blockIdx.x * 4 + (threadIdx.x >> 6) : blockIdx.x;
  if (unit >= units) return;                        // whole wave or block
  const long long row = unit / parts;
  const int c0 = (int)(unit % parts) * n;
  const T* xr = x + row * parts * n + c0;
  T* orow = out + row * ostride + c0;
  float ss = 0.f;
  for (int i = tid * VEC; i < n; i += nth * VEC) {
    float v[VEC];
    ldv<T, VEC>(xr + i, v);
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss = fmaf(v[j], v[j], ss);
  }
  ss = WAVE ? wave_reduce_sum(ss) : block_reduce_sum(ss, scratch);
  const float inv = 1.f / sqrtf(ss / (float)n + eps);
  for (int i = tid * VEC; i < n; i += nth * VEC) {
    float v[VEC], wv[VEC];
    ldv<T, VEC>(xr + i, v);
    ldv<float, VEC>(w + c0 + i, wv);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] *= inv * wv[j];
    stv<T, VEC>(orow + i, v);
  }
}

extern "C" void qsa_part_norm_launch(const void* x, const float* w, void* out,
                                     long long ostride, long long rows,
                                     int parts, int n, float eps, int f32,
                                     int vec, hipStream_t st) {
  const long long units = rows * parts;
  const bool wave = n <= (vec ? 1024 : 256);
  const long long blocks = wave ? (units + 3) / 4 : units;
#define QSA_PN(T, V, W)                                                      \
  hipLaunchKernelGGL((qsa_part_norm<T, V, W>), dim3((unsigned)blocks),       \
                     dim3(256), 0, st, (const T*)x, w, (T*)out, ostride,     \
                     units, parts, n, eps)
  if (f32) {
    if (vec) { if (wave) QSA_PN(float, 4, true); else QSA_PN(float, 4, false); }
    else     { if (wave) QSA_PN(float, 1, true); else QSA_PN(float, 1, false); }
  } else {
    if (vec) { if (wave) QSA_PN(bf16_t, 4, true); else QSA_PN(bf16_t, 4, false); }
    else     { if (wave) QSA_PN(bf16_t, 1, true); else QSA_PN(bf16_t, 1, false); }
  }
#undef QSA_PN
}
