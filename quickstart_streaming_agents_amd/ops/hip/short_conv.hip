// Short causal convolutions over time, one filter per channel:
//   y_t[c] = bias[c] + sum_j w[j][c] u_(t - taps + 1 + j)[c]
// u are columns of a projected row; zeros stand before a sequence's first
// token, and the last taps - 1 inputs of every sequence are its tail:
// tails [slots, taps - 1, C] in the storage type, oldest first.
//
// A thread owns a few channels for CONV_ROWS tokens of one portion (its window
// stays in registers).  Only the first tokens of a portion look at the old
// tail, and the thread that owns them also writes the new one, so reading and
// writing it never race.  Tail entries before position 0 read as zero: slots
// need no clearing between owners.
//
//   qsa_conv_qkv   channels [q | k | v] of an attention layer, then the
//                  rotation of q and k; k and v go straight to their pages
//   qsa_conv_silu  bias and silu, to a dense [rows, C]
#include "lm_common.h"

#define CONV_ROWS 16  // tokens per thread; taps - 1 must not exceed it

struct ConvStep {
  const int* item;   // portion of a chunk of rows; null: chunk c is row c,
  const int* t0;     //   one token at position start[c] - 1
  const int* off;
  const int* start;
  const int* len;
  const int* slots;
};

struct ConvSpan { int r0, t0, t1, n, p0, slot; };

__device__ __forceinline__ ConvSpan conv_span(const ConvStep& st, int c) {
  ConvSpan s;
  if (st.item) {
    const int it = st.item[c];
    s.r0 = st.off[it];
    s.t0 = st.t0[c];
    s.n = st.len[it];
    s.p0 = st.start[it];
    s.slot = st.slots[it];
    s.t1 = min(s.t0 + CONV_ROWS, s.n);
  } else {
    s.r0 = c;
    s.t0 = 0;
    s.n = s.t1 = 1;
    s.p0 = st.start[c] - 1;
    s.slot = st.slots[c];
  }
  return s;
}

// NP (1 or 2) groups of VEC channels, c0.. and c1..; TAPS 0: `taps` of them,
// through memory.  pre(t) loads what emit(t, values, .) wants besides.
template <typename T, int TAPS, int VEC, int NP, typename Pre, typename Emit>
__device__ __forceinline__ void conv_rows(
    const T* x, long long xstride, T* tail, int C, int c0, int c1,
    const float* w, const float* bias, int taps, const ConvSpan& s, Pre pre,
    Emit emit) {
  const int NT = (TAPS ? TAPS : taps) - 1;
  auto ch = [&](int p) { return p == 0 ? c0 : c1; };
  auto load = [&](int t, int p, float* v) {
    if (t >= 0) {
      ldv<T, VEC>(x + (long long)(s.r0 + t) * xstride + ch(p), v);
    } else if (s.p0 + t >= 0) {
      ldv<T, VEC>(tail + (long long)(NT + t) * C + ch(p), v);
    } else {
#pragma unroll
      for (int i = 0; i < VEC; ++i) v[i] = 0.f;
    }
  };
  float b[NP][VEC];
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    if (bias) {
      ldv<float, VEC>(bias + ch(p), b[p]);
    } else {
#pragma unroll
      for (int i = 0; i < VEC; ++i) b[p][i] = 0.f;
    }
  }
  if constexpr (TAPS > 0) {
    constexpr int K = TAPS > 1 ? TAPS - 1 : 1;
    float wt[NP][TAPS][VEC], win[NP][K][VEC];
#pragma unroll
    for (int p = 0; p < NP; ++p) {
#pragma unroll
      for (int j = 0; j < TAPS; ++j)
        ldv<float, VEC>(w + (long long)j * C + ch(p), wt[p][j]);
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j)
        load(s.t0 - (TAPS - 1) + j, p, win[p][j]);
    }
#pragma unroll 4
    for (int t = s.t0; t < s.t1; ++t) {
      const auto aux = pre(t);
      float a[NP][VEC];
#pragma unroll
      for (int p = 0; p < NP; ++p) {
        float u[VEC];
        ldv<T, VEC>(x + (long long)(s.r0 + t) * xstride + ch(p), u);
#pragma unroll
        for (int i = 0; i < VEC; ++i) {
          a[p][i] = b[p][i];
#pragma unroll
          for (int j = 0; j < TAPS - 1; ++j)
            a[p][i] = fmaf(wt[p][j][i], win[p][j][i], a[p][i]);
          a[p][i] = fmaf(wt[p][TAPS - 1][i], u[i], a[p][i]);
#pragma unroll
          for (int j = 0; j + 2 < TAPS; ++j) win[p][j][i] = win[p][j + 1][i];
          win[p][K - 1][i] = u[i];
        }
      }
      emit(t, a, aux);
    }
  } else {
    for (int t = s.t0; t < s.t1; ++t) {
      const auto aux = pre(t);
      float a[NP][VEC];
#pragma unroll
      for (int p = 0; p < NP; ++p) {
#pragma unroll
        for (int i = 0; i < VEC; ++i) a[p][i] = b[p][i];
        for (int j = 0; j <= NT; ++j) {
          float u[VEC], wj[VEC];
          load(t - NT + j, p, u);
          ldv<float, VEC>(w + (long long)j * C + ch(p), wj);
#pragma unroll
          for (int i = 0; i < VEC; ++i) a[p][i] = fmaf(wj[i], u[i], a[p][i]);
        }
      }
      emit(t, a, aux);
    }
  }
  if (s.t0 == 0) {
    // entry j moves from n + j, never from a place already overwritten
    for (int j = 0; j < NT; ++j)
#pragma unroll
      for (int p = 0; p < NP; ++p) {
        float v[VEC];
        load(s.n - NT + j, p, v);
        stv<T, VEC>(tail + (long long)j * C + ch(p), v);
      }
  }
}

#define CONV_CASE(T, TAPS, VEC, NP)                                          \
  conv_rows<T, TAPS, VEC, NP>(x, xstride, tail, C, c0, c1, w, bias, taps, s, \
                              pre, emit)
#define CONV_DISPATCH(T, VEC, NP)              \
  switch (taps) {                              \
    case 1: CONV_CASE(T, 1, VEC, NP); break;   \
    case 2: CONV_CASE(T, 2, VEC, NP); break;   \
    case 3: CONV_CASE(T, 3, VEC, NP); break;   \
    case 4: CONV_CASE(T, 4, VEC, NP); break;   \
    default: CONV_CASE(T, 0, VEC, NP);         \
  }

template <int VEC>
struct Turn {
  int slot;                    // where k or v goes
  float c[VEC], s[VEC];
};

// A thread owns a pair of channel groups: of q and k a rotated pair (i,
// i + rot/2) or two groups behind the rotated ones, of v two groups.
// Pages: k [pages, G, 64, D], v [pages, G, 64, E].
template <typename T, int VEC>
__global__ void __launch_bounds__(256)
qsa_conv_qkv(const T* x, long long xstride, const float* __restrict__ w,
             int taps, T* tails, ConvStep step,
             const float* __restrict__ cos_t, const float* __restrict__ sin_t,
             int rot, int table_len, const int* __restrict__ cache_slots,
             T* __restrict__ q, T* __restrict__ kc, T* __restrict__ vc, int H,
             int G, int D, int E) {
  const int half = rot >> 1;
  const int ur = half / VEC, up = (D - rot + 2 * VEC - 1) / (2 * VEC);
  const int ud = ur + up, ue = (E + 2 * VEC - 1) / (2 * VEC);
  const int u = blockIdx.y * blockDim.x + threadIdx.x;
  if (u >= (H + G) * ud + G * ue) return;
  const ConvSpan s = conv_span(step, blockIdx.x);
  if (s.slot < 0 || s.p0 < 0) return;
  const int C = (H + G) * D + G * E;
  T* tail = tails + (long long)s.slot * (taps - 1) * C;
  const float* bias = nullptr;
  const bool val = u >= (H + G) * ud;
  const int un = val ? ue : ud;
  const int r = (val ? u - (H + G) * ud : u) % un;
  const int head = (val ? u - (H + G) * ud : u) / un;
  const bool turn = !val && r < ur;
  const int d0 = val || turn ? r * VEC : rot + (r - ur) * VEC;
  const int far = d0 + (val ? ue * VEC : turn ? half : up * VEC);
  const bool two = far < (val ? E : D);
  const int d1 = two ? far : d0;
  const int base = val ? (H + G) * D + head * E : head * D;
  const int c0 = base + d0, c1 = base + d1;
  const bool query = !val && head < H;
  auto pre = [=](int t) {
    Turn<VEC> r;
    r.slot = query ? 0 : cache_slots[s.r0 + t];
    if (turn) {
      const long long at =
          (long long)min(s.p0 + t, table_len - 1) * half + d0;
      ldv<float, VEC>(cos_t + at, r.c);
      ldv<float, VEC>(sin_t + at, r.s);
    }
    return r;
  };
  auto emit = [=](int t, float (&a)[2][VEC], const Turn<VEC>& r) {
    const long long row = s.r0 + t;
    if (turn) {
#pragma unroll
      for (int i = 0; i < VEC; ++i) {
        const float u0 = a[0][i], v0 = a[1][i];
        a[0][i] = u0 * r.c[i] - v0 * r.s[i];
        a[1][i] = v0 * r.c[i] + u0 * r.s[i];
      }
    }
    T* dst;
    if (query) {
      dst = q + (row * H + head) * D;
    } else {
      if (r.slot < 0) return;
      const long long at = (long long)(r.slot >> 6) * G +
                           (val ? head : head - H);
      dst = val ? vc + (at * 64 + (r.slot & 63)) * E
                : kc + (at * 64 + (r.slot & 63)) * D;
    }
    stv<T, VEC>(dst + d0, a[0]);
    if (two) stv<T, VEC>(dst + d1, a[1]);
  };
  CONV_DISPATCH(T, VEC, 2)
}

extern "C" void qsa_conv_qkv_launch(
    const void* x, long long xstride, const float* w, int taps, void* tails,
    ConvStep step, int chunks, const float* cos_t, const float* sin_t,
    int rot, int table_len, const int* cache_slots, void* q, void* kc,
    void* vc, int H, int G, int D, int E, int f32, int vec4, hipStream_t st) {
  const int V = vec4 ? 4 : 1;
  const int ud = (rot / 2) / V + (D - rot + 2 * V - 1) / (2 * V);
  const int units = (H + G) * ud + G * ((E + 2 * V - 1) / (2 * V));
  const int threads = units <= 64 ? 64 : units <= 128 ? 128 : 256;
  dim3 grid((unsigned)chunks, (unsigned)((units + threads - 1) / threads));
#define QSA_CQ(T, V)                                                         \
  hipLaunchKernelGGL((qsa_conv_qkv<T, V>), grid, dim3(threads), 0, st,       \
                     (const T*)x, xstride, w, taps, (T*)tails, step, cos_t,  \
                     sin_t, rot, table_len, cache_slots, (T*)q, (T*)kc,      \
                     (T*)vc, H, G, D, E)
  if (f32) { if (vec4) QSA_CQ(float, 4); else QSA_CQ(float, 1); }
  else     { if (vec4) QSA_CQ(bf16_t, 4); else QSA_CQ(bf16_t, 1); }
#undef QSA_CQ
}

template <typename T, int VEC>
__global__ void __launch_bounds__(256)
qsa_conv_silu(const T* x, long long xstride, const float* __restrict__ w,
              const float* __restrict__ bias, int taps, T* tails,
              ConvStep step, T* __restrict__ out, int C) {
  const int u = blockIdx.y * blockDim.x + threadIdx.x;
  if (u >= C / VEC) return;
  const ConvSpan s = conv_span(step, blockIdx.x);
  if (s.slot < 0 || s.p0 < 0) return;
  T* tail = tails + (long long)s.slot * (taps - 1) * C;
  const int c0 = u * VEC, c1 = c0;
  auto pre = [](int) { return 0; };
  auto emit = [=](int t, float (&a)[1][VEC], int) {
#pragma unroll
    for (int i = 0; i < VEC; ++i)
      a[0][i] = sizeof(T) == 4 ? silu_f(a[0][i])
                               : a[0][i] / (1.f + __expf(-a[0][i]));
    stv<T, VEC>(out + (long long)(s.r0 + t) * C + c0, a[0]);
  };
  CONV_DISPATCH(T, VEC, 1)
}

extern "C" void qsa_conv_silu_launch(const void* x, long long xstride,
                                     const float* w, const float* bias,
                                     int taps, void* tails, ConvStep step,
                                     int chunks, void* out, int C, int f32,
                                     int vec4, hipStream_t st) {
  const int units = vec4 ? C / 4 : C;
  const int threads = units <= 64 ? 64 : units <= 128 ? 128 : 256;
  dim3 grid((unsigned)chunks, (unsigned)((units + threads - 1) / threads));
#define QSA_CS(T, V)                                                        \
  hipLaunchKernelGGL((qsa_conv_silu<T, V>), grid, dim3(threads), 0, st,     \
                     (const T*)x, xstride, w, bias, taps, (T*)tails, step,  \
                     (T*)out, C)
  if (f32) { if (vec4) QSA_CS(float, 4); else QSA_CS(float, 1); }
  else     { if (vec4) QSA_CS(bf16_t, 4); else QSA_CS(bf16_t, 1); }
#undef QSA_CS
}
