// Products of float rows with weights of the compute dtype on the matrix cores, for the small matrices
// whose results enter a recurrence: the rows are not rounded.
#pragma once
#include "common.h"

// Sixteen rows times NT x 16 features, for one wave.  `x(k)` gives the float4 at columns k .. k + 3 (k a
// multiple of 4) of row lane % 16; w[j] is the row of weights (K of them, K a multiple of 8, 16-byte
// aligned) of feature 16 j + lane % 16.  acc[j] holds, as D of v_mfma_f32_16x16*: rows 4 (lane / 16) + i,
// feature 16 j + lane % 16.  The wave takes the pieces of 32 columns `first`, `first + step`, ...
//   bfloat16 weights: a float is the sum of a bfloat16 and a bfloat16 of what is left, two
//   v_mfma_f32_16x16x32_bf16 a tile (16 bits of the row's float count).
//   float weights: v_mfma_f32_16x16x4_f32, lanes bring four consecutive columns to four instructions.
union RowsFrag {
  u32x4_t u;
  bf16x8_t v;
};
// One piece of 32 columns from k on (this lane's are k + 8 (lane / 16) ..): b are the weights' fragments.
template <int NT, typename Rows>
__device__ __forceinline__ void rows_piece(Rows x, const RowsFrag (&b)[NT], int K, int k0, f32x4_t (&acc)[NT]) {
  const int k = k0 + 8 * ((threadIdx.x & 63) >> 4);
  const bool in = k < K;
  float f[8];
  *(float4*)f = x(in ? k : 0), *(float4*)(f + 4) = x(in ? k + 4 : 4);
  RowsFrag hi, lo;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float a = in ? f[2 * i] : 0.f, c = in ? f[2 * i + 1] : 0.f;
    hi.u[i] = pack_bf16x2(a, c);
    lo.u[i] = pack_bf16x2(a - bits_to_f32((uint16_t)(hi.u[i] & 0xffffu)), c - bits_to_f32((uint16_t)(hi.u[i] >> 16)));
  }
#pragma unroll
  for (int j = 0; j < NT; ++j) {
    acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi.v, b[j].v, acc[j], 0, 0, 0);
    acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo.v, b[j].v, acc[j], 0, 0, 0);
  }
}
template <int NT>
__device__ __forceinline__ void ask_piece(const bf16* const (&w)[NT], int K, int k0, RowsFrag (&b)[NT]) {
  const int k = k0 + 8 * ((threadIdx.x & 63) >> 4);
#pragma unroll
  for (int j = 0; j < NT; ++j) b[j].u = *(const u32x4_t*)(w[j] + (k < K ? k : 0));
}

template <int NT, typename Rows>
__device__ __forceinline__ void rows_product(Rows x, const bf16* const (&w)[NT], int K, int first, int step, f32x4_t (&acc)[NT]) {
  if (32 * first >= K) return;
  RowsFrag b[NT], next[NT];
  ask_piece<NT>(w, K, 32 * first, b);
  for (int k0 = 32 * first; k0 < K; k0 += 32 * step) {
    ask_piece<NT>(w, K, k0 + 32 * step, next);  // (a piece ahead; behind the last one the first columns again)
    rows_piece<NT>(x, b, K, k0, acc);
#pragma unroll
    for (int j = 0; j < NT; ++j) b[j] = next[j];
  }
}

// The first PIECES pieces' weights, to be asked for before the rows are known.
template <int NT, int PIECES>
struct PiecesAhead {
  RowsFrag b[PIECES][NT];
  __device__ __forceinline__ void ask(const bf16* const (&w)[NT], int K, int first, int step) {
#pragma unroll
    for (int i = 0; i < PIECES; ++i) ask_piece<NT>(w, K, 32 * (first + i * step), b[i]);
  }
  template <typename Rows>
  __device__ __forceinline__ void product(Rows x, int K, int first, int step, f32x4_t (&acc)[NT]) {
#pragma unroll
    for (int i = 0; i < PIECES; ++i)
      if (32 * (first + i * step) < K) rows_piece<NT>(x, b[i], K, 32 * (first + i * step), acc);
  }
};

template <int NT, typename Rows>
__device__ __forceinline__ void rows_product(Rows x, const float* const (&w)[NT], int K, int first, int step, f32x4_t (&acc)[NT]) {
  const int g = (threadIdx.x & 63) >> 4;
  for (int k0 = 32 * first; k0 < K; k0 += 32 * step) {
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      const int k = k0 + 16 * half + 4 * g;
      const bool in = k < K;
      const float4 v = x(in ? k : 0);
      const float f[4] = {in ? v.x : 0.f, in ? v.y : 0.f, in ? v.z : 0.f, in ? v.w : 0.f};
#pragma unroll
      for (int j = 0; j < NT; ++j) {
        const float4 b = *(const float4*)(w[j] + (in ? k : 0));
        acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(f[0], b.x, acc[j], 0, 0, 0);
        acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(f[1], b.y, acc[j], 0, 0, 0);
        acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(f[2], b.z, acc[j], 0, 0, 0);
        acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(f[3], b.w, acc[j], 0, 0, 0);
      }
    }
  }
}
