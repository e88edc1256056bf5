// Shared device helpers of the decoder-mixer kernels (qsa_lm_hip).
//
// Every scalar kernel is a template over the storage type T: bf16 (held as
// unsigned short) or float.  All arithmetic is f32; T is only how operands
// and results are stored.
#pragma once

#include "common.h"

typedef unsigned short bf16_t;

using bf16x8_v = __attribute__((ext_vector_type(8))) short;
using bf16x4_v = __attribute__((ext_vector_type(4))) short;
using u32x4_v = __attribute__((ext_vector_type(4))) unsigned int;
using f32x4_v = __attribute__((ext_vector_type(4))) float;

// round-to-nearest-even with the hardware's packed conversion
__device__ __forceinline__ unsigned int cvt_bf16x2(float a, float b) {
  typedef __attribute__((ext_vector_type(2))) float f2;
  typedef __attribute__((ext_vector_type(2))) __bf16 b2;
  return __builtin_bit_cast(unsigned int,
                            __builtin_convertvector((f2){a, b}, b2));
}
__device__ __forceinline__ bf16_t cvt_bf16(float a) {
  return __builtin_bit_cast(bf16_t, (__bf16)a);
}

template <typename T> __device__ __forceinline__ float ldf(const T* p);
template <> __device__ __forceinline__ float ldf<bf16_t>(const bf16_t* p) {
  return bf16_to_f32(*p);
}
template <> __device__ __forceinline__ float ldf<float>(const float* p) {
  return *p;
}
template <typename T> __device__ __forceinline__ void stf(T* p, float v);
template <> __device__ __forceinline__ void stf<bf16_t>(bf16_t* p, float v) {
  *p = cvt_bf16(v);
}
template <> __device__ __forceinline__ void stf<float>(float* p, float v) {
  *p = v;
}

// VEC consecutive elements <-> f32 registers (pointer aligned to the group)
template <typename T, int VEC>
__device__ __forceinline__ void ldv(const T* p, float* v) {
  if constexpr (VEC == 1) {
    v[0] = ldf<T>(p);
  } else if constexpr (sizeof(T) == 4) {
#pragma unroll
    for (int i = 0; i < VEC; i += 4) {
      const float4 f = *reinterpret_cast<const float4*>(p + i);
      v[i] = f.x; v[i + 1] = f.y; v[i + 2] = f.z; v[i + 3] = f.w;
    }
  } else {
#pragma unroll
    for (int i = 0; i < VEC; i += 4) {
      const uint2 u = *reinterpret_cast<const uint2*>(p + i);
      const float2 a = bf16x2_to_f32x2(u.x), b = bf16x2_to_f32x2(u.y);
      v[i] = a.x; v[i + 1] = a.y; v[i + 2] = b.x; v[i + 3] = b.y;
    }
  }
}
template <typename T, int VEC>
__device__ __forceinline__ void stv(T* p, const float* v) {
  if constexpr (VEC == 1) {
    stf<T>(p, v[0]);
  } else if constexpr (sizeof(T) == 4) {
#pragma unroll
    for (int i = 0; i < VEC; i += 4)
      *reinterpret_cast<float4*>(p + i) =
          make_float4(v[i], v[i + 1], v[i + 2], v[i + 3]);
  } else {
#pragma unroll
    for (int i = 0; i < VEC; i += 4)
      *reinterpret_cast<uint2*>(p + i) = make_uint2(
          cvt_bf16x2(v[i], v[i + 1]), cvt_bf16x2(v[i + 2], v[i + 3]));
  }
}

__device__ __forceinline__ float silu_f(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float sigmoid_f(float z) {
  return 1.f / (1.f + expf(-z));
}

// x = hi + lo with both parts bf16: 16 mantissa bits survive, so a product
// of two such pairs on the bf16 matrix cores (hi*hi + hi*lo + lo*hi) stays
// at f32-like accuracy.
__device__ __forceinline__ void split_bf16(float x, bf16_t& hi, bf16_t& lo) {
  hi = cvt_bf16(x);
  lo = cvt_bf16(x - bf16_to_f32(hi));
}

// four values -> their packed hi and lo parts
__device__ __forceinline__ void split4_bf16(float a, float b, float c, float d,
                                            uint2& hi, uint2& lo) {
  hi = make_uint2(cvt_bf16x2(a, b), cvt_bf16x2(c, d));
  const float2 h0 = bf16x2_to_f32x2(hi.x), h1 = bf16x2_to_f32x2(hi.y);
  lo = make_uint2(cvt_bf16x2(a - h0.x, b - h0.y),
                  cvt_bf16x2(c - h1.x, d - h1.y));
}

// Barrier that orders LDS accesses only: global loads and stores in flight
// stay in flight (their users wait for the registers).
__device__ __forceinline__ void lds_barrier() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
  __builtin_amdgcn_s_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
}

// Transposing LDS read: within 16 lanes, lane i supplies the address of 4
// consecutive elements of row i/4, columns (i%4)*4.. of a 4 x 16 block and
// receives column i, i.e. 4 consecutive rows of one column.
__device__ __forceinline__ bf16x4_v lds_read_tr(const bf16_t* p) {
  typedef __attribute__((address_space(3))) bf16x4_v* lds_ptr;
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)p);
}

// Two transposed 4-row groups of column `col_tile*16 + lane%16` as one
// 8-element MFMA operand: rows row0 + hi*4 .. +3 and row1 + hi*4 .. +3
// (hi = lane / 16).
__device__ __forceinline__ bf16x8_v lds_frag_tr(const bf16_t* tile, int pitch,
                                                int row0, int row1, int col0,
                                                int lane) {
  const int r = (lane >> 4) * 4 + ((lane & 15) >> 2);
  const int c = col0 + (lane & 3) * 4;
  const bf16x4_v a = lds_read_tr(tile + (row0 + r) * pitch + c);
  const bf16x4_v b = lds_read_tr(tile + (row1 + r) * pitch + c);
  return __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
}

__device__ __forceinline__ f32x4_v mfma_bf16(bf16x8_v a, bf16x8_v b,
                                             f32x4_v c) {
  typedef __attribute__((ext_vector_type(8))) __bf16 raw;
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(
      __builtin_bit_cast(raw, a), __builtin_bit_cast(raw, b), c, 0, 0, 0);
}
