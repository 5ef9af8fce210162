// Device code shared by the recurrent mixers whose kernels read projected rows themselves (fixed_decay.hip,
// matrix_memory.hip).
#pragma once
#include "common.h"

typedef __attribute__((ext_vector_type(4))) float f32x4;

__device__ __forceinline__ float recurrent_act(float z, int silu) { return silu ? z / (1.0f + expf(-z)) : z; }

// four numbers of a projected row from feature i on (those at or beyond `end` are zero), activated
template <typename T>
__device__ __forceinline__ void load_row4(const T* row, int i, int end, bool vec, int silu, float (&v)[4]) {
  if (vec && i + 4 <= end) {
    if (sizeof(T) == 4) {
      const float4 x = *reinterpret_cast<const float4*>((const float*)row + i);
      v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w;
    } else {
      const uint2 x = *reinterpret_cast<const uint2*>((const bf16_t*)row + i);  // a bfloat16 is the upper half of a float
      v[0] = __uint_as_float(x.x << 16); v[1] = __uint_as_float(x.x & 0xffff0000u);
      v[2] = __uint_as_float(x.y << 16); v[3] = __uint_as_float(x.y & 0xffff0000u);
    }
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = i + e < end ? to_f32(row[i + e]) : 0.f;
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = recurrent_act(v[e], silu);  // SiLU of 0 is 0
}

// Sum over 16 neighbouring lanes, in every one of them.
__device__ __forceinline__ float sum16(float v) {
  v += __shfl_xor(v, 8, 16);
  v += __shfl_xor(v, 4, 16);
  v += __shfl_xor(v, 2, 16);
  v += __shfl_xor(v, 1, 16);
  return v;
}
