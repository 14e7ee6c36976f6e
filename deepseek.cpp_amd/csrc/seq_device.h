// seq_device.h -- device pieces shared by the kernels of layered models: activation types, matrix fragments, reductions.
//
// Activations are T = bf16 or float; weights are always bf16 in HBM (a 32-bit run multiplies their exact values).  Every matrix
// lives as FRAGMENTS of 16 rows x 32 columns: 64 lanes x 8 consecutive k, lane = (k / 8) * 16 + row, 1 KiB contiguous - the
// operand order of v_mfma_f32_16x16x32_bf16.  A wave reads a fragment with one 16-byte load per lane from consecutive
// addresses, in HBM and in LDS alike.  A 32-bit run multiplies the same fragments with eight v_mfma_f32_16x16x4_f32: step j
// takes element j of every lane, so lane groups stand for the k values {8 g + j}.
#pragma once
#include "dsk_internal.h"

typedef __bf16 bf16;
typedef bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x8 __attribute__((ext_vector_type(8)));
#define DEV __device__ __forceinline__

template <typename T>
struct Frag;
template <>
struct Frag<bf16> {
  typedef bf16x8 type;
  typedef bf16x4 four;
};
template <>
struct Frag<float> {
  typedef f32x8 type;
  typedef f32x4 four;
};

DEV f32x4 mma(const bf16x8& w, const bf16x8& a, const f32x4& c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(w, a, c, 0, 0, 0); }
DEV f32x4 mma(const bf16x8& w, const f32x8& a, f32x4 c) {
#pragma unroll
  for (int j = 0; j < 8; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32((float)w[j], a[j], c, 0, 0, 0);
  return c;
}
DEV f32x4 mma(const f32x8& w, const f32x8& a, f32x4 c) {
#pragma unroll
  for (int j = 0; j < 8; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(w[j], a[j], c, 0, 0, 0);
  return c;
}

// A block of 16 rows x 32 columns on its way from row-major memory to operands: loaded row by row, four lanes to a row, lane l's 8 columns
// at place l of the block in LDS.  Inside a row the groups are exchanged by the row's place, so that the lanes that read one group of 16 rows
// meet every LDS bank once.
DEV int block_row(int lane) { return lane >> 2; }                                              // what lane l loads ...
DEV int block_group(int lane) { return (lane & 3) ^ (lane >> 4); }
DEV int block_place(int lane) { return (lane & 15) * 4 + ((lane >> 4) ^ ((lane >> 2) & 3)); }  // ... and the place that lane l of an operand reads

template <typename T>
DEV typename Frag<T>::four to_four(const f32x4& v) {
  return __builtin_convertvector(v, typename Frag<T>::four);
}

// a barrier for LDS traffic only: global loads and stores stay in flight across it (__syncthreads drains them)
DEV void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

DEV float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }
DEV float silu_f(float x) { return x * sigmoid_f(x); }
DEV float softplus_f(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
DEV float logsigmoid_f(float x) { return -softplus_f(-x); }

DEV float wave_sum(float v) {
#pragma unroll
  for (int off = 32; off >= 1; off >>= 1) v += __shfl_xor(v, off);
  return v;
}
// sum over a row of 16 lanes, result in all of them: four DPP adds
template <int CTRL>
DEV float dpp_f(float v) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
DEV float row_sum(float v) {
  v += dpp_f<0xB1>(v);   // quad_perm [1, 0, 3, 2]
  v += dpp_f<0x4E>(v);   // quad_perm [2, 3, 0, 1]
  v += dpp_f<0x141>(v);  // row_half_mirror
  v += dpp_f<0x140>(v);  // row_mirror
  return v;
}
// sum over a workgroup of NT threads, result in every thread; scratch: NT / 64 floats of LDS
template <int NT>
DEV float block_sum(float v, float* scratch) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < NT / 64; ++i) s += scratch[i];
  return s;
}
