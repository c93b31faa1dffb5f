// Device helpers the kernels of hybrid decoders share: rotary angles, reductions, swizzled LDS tiles filled by
// LDS-direct loads, fp32 matrix instructions.
#pragma once

#include "skinny.cuh"

namespace mui {

// cos and sin of pos * inv_freq: the angle in turns, its whole turns dropped in double precision, rounded once
__device__ __forceinline__ void rope_angle(double pos, double inv_freq, float& c, float& s) {
  double a = pos * inv_freq * 0.15915494309189533576888376337251;
  a -= rint(a);
  sincospif((float)(2.0 * a), &s, &c);
}

__device__ __forceinline__ float block_sum256(float v, float* red) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & (kWave - 1)) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return (red[0] + red[1]) + (red[2] + red[3]);
}

// LDS tiles filled by LDS-direct loads: blocks of 64 columns, in a block rows of 128 bytes whose 16-byte chunk c
// lives at chunk c ^ ((row >> 1) & 7) (16 rows of one logical chunk fall into 64 different banks). A wave
// instruction delivers eight rows of one block.
__device__ __forceinline__ int tile_swz(int row) { return (row >> 1) & 7; }
template <int ROWS>
__device__ __forceinline__ int tile_at(int row, int col) {  // in elements
  return ((col >> 6) * ROWS + row) * 64 + ((((col >> 3) & 7) ^ tile_swz(row)) << 3) + (col & 7);
}

// v_mfma_f32_16x16x4_f32 (A: row lane % 16, k lane / 16; B: column lane % 16; D: column lane % 16, rows 4 (lane / 16) + r)
__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

}  // namespace mui
