// Helpers shared by the kernels behind include/e2h_seq.h.
#pragma once

#include "../../include/e2h_seq.h"
#include "e2h_common.h"

namespace e2h {

struct SeqOptions {
  int recurrence_form;         // 0 = by token count, 1 = token by token, 2 = chunked
  int recurrence_chunk;        // 0 = heuristic, else tokens per workgroup of the chunked HGRN2 form (multiple of 16)
  int norm_run;                // 0 = heuristic, else tokens per workgroup of the norm kernel
  int attention_decode_waves;  // 0 = by window, else 4 or 8
  int attention_query_tiles;   // 0 = by token count, else 1 or 2 tiles of 16 queries per wave
};
SeqOptions &seq_options();

// typed loads and stores: bf16_t holds a bfloat16 bit pattern
typedef uint16_t bf16_t;

__device__ __forceinline__ float to_f32(bf16_t v) { return bf16_to_f32(v); }
__device__ __forceinline__ float to_f32(float v) { return v; }
template <typename T>
__device__ __forceinline__ T from_f32(float v);
template <>
__device__ __forceinline__ bf16_t from_f32<bf16_t>(float v) {
  return f32_to_bf16_rne(v);
}
template <>
__device__ __forceinline__ float from_f32<float>(float v) {
  return v;
}

__device__ __forceinline__ f32x4_t load4(const float *p) { return *reinterpret_cast<const f32x4_t *>(p); }
__device__ __forceinline__ f32x4_t load4(const bf16_t *p) {
  const u32x2_t r = *reinterpret_cast<const u32x2_t *>(p);
  return f32x4_t{__builtin_bit_cast(float, r[0] << 16), __builtin_bit_cast(float, r[0] & 0xFFFF0000u), __builtin_bit_cast(float, r[1] << 16),
                 __builtin_bit_cast(float, r[1] & 0xFFFF0000u)};
}
__device__ __forceinline__ void store4(float *p, f32x4_t v) { *reinterpret_cast<f32x4_t *>(p) = v; }
__device__ __forceinline__ void store4(bf16_t *p, f32x4_t v) {
  u32x2_t r;
  r[0] = static_cast<uint32_t>(f32_to_bf16_rne(v[0])) | (static_cast<uint32_t>(f32_to_bf16_rne(v[1])) << 16);
  r[1] = static_cast<uint32_t>(f32_to_bf16_rne(v[2])) | (static_cast<uint32_t>(f32_to_bf16_rne(v[3])) << 16);
  *reinterpret_cast<u32x2_t *>(p) = r;
}

__device__ __forceinline__ float wave_add(float v) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off);
  return v;
}

constexpr float kLog2e = 1.4426950408889634f;

// acc += A B over 16 rows of B in four steps of v_mfma_f32_16x16x4_f32.  Lane (b, c) = 16 b + c gives A[c][4 b .. 4 b + 3] and
// B[4 b .. 4 b + 3][c]: step r multiplies rows {4 b + r}, so B may be the accumulators of another product as they are.
__device__ __forceinline__ f32x4_t mfma4(f32x4_t a, f32x4_t b, f32x4_t acc) {
#pragma unroll
  for (int r = 0; r < 4; ++r) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[r], b[r], acc, 0, 0, 0);
  return acc;
}

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f32(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }

}  // namespace e2h
