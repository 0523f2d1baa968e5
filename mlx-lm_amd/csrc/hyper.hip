// Hyper-connections: a residual stream that is kept as S streams.  A sublayer reads a weighted sum of
// them, u = sum_s in[s] x_s, and its output y enters all of them at once,
//   x_t <- sum_s mix[s][t] x_s + out[t] y      (mix is indexed [from][to])
// Between two sublayers one kernel does all there is: the write behind the first (y may still lie in
// the parts in which a product left it), the read ahead of the second and that one's norm.
//
//   hyper_step   a block a token, the streams of a token side by side ([tokens, S, D]):
//                  x_s = xs[s], or all of them `first` (the embedding's rows) where xs is null
//                  with y: the write;  xs_out (may be xs itself): the new streams
//                  u = sum_s in[s] x_s (in null: the plain sum)
//                  norm_out = LayerNorm(u) * gamma + beta, and/or sum_out = u
//                  rows_out = W norm_out for a small matrix W (a router's): a step of few tokens saves the
//                  launch that this product would be
// All 32-bit; only norm_out may be bfloat16.
#include "common.h"

#define MAX_STREAMS 8
#define MAX_ROWS 128  // of the small matrix

struct HyperArgs {
  const float* xs;
  const float* first;
  int ld_first;
  float* xs_out;
  const float* y;  // n_parts of [T, D], rows of stride ldy, parts y_part floats apart
  int ldy, n_parts;
  size_t y_part;
  const float* bias;  // [D], added to y with its parts, or null
  const float* mix;   // [S][S]
  const float* out;   // [S]
  const float* in;    // [S]
  const float* gamma;
  const float* beta;
  float eps;
  void* norm_out;  // [T, D]
  int norm_dtype;
  float* sum_out;
  int ld_sum;
  int T, D, S;
  const void* w;  // [n_rows][D] of norm_out's dtype, or null
  float* rows_out;  // [T, n_rows]
  int n_rows;
};

__device__ __forceinline__ f32x4_t four(const bf16* p) {
  const uint2 v = *(const uint2*)p;
  return f32x4_t{__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u), __uint_as_float(v.y << 16), __uint_as_float(v.y & 0xffff0000u)};
}
__device__ __forceinline__ f32x4_t four(const float* p) { return *(const f32x4_t*)p; }

// rows_out[t] = W u for the normed row that the block's threads hold (u[i]: columns 4 (tid + TH i) ..)
template <typename T, int NV, int TH>
__device__ __forceinline__ void small_rows(const HyperArgs& a, int t, const f32x4_t (&u)[NV], float (*part)[MAX_ROWS]) {
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const T* w = (const T*)a.w;
  for (int e0 = 0; e0 < a.n_rows; e0 += 8) {
    f32x4_t wv[8][NV];
#pragma unroll
    for (int e = 0; e < 8; ++e)
#pragma unroll
      for (int i = 0; i < NV; ++i) wv[e][i] = four(w + (size_t)min(e0 + e, a.n_rows - 1) * a.D + min(4 * (tid + TH * i), a.D - 4));
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      float s = 0.f;
#pragma unroll
      for (int i = 0; i < NV; ++i)
        if (4 * (tid + TH * i) < a.D) s += (wv[e][i][0] * u[i][0] + wv[e][i][1] * u[i][1]) + (wv[e][i][2] * u[i][2] + wv[e][i][3] * u[i][3]);
      s = wave_sum(s);
      if (lane == 0 && e0 + e < a.n_rows) part[wave][e0 + e] = s;
    }
  }
  __syncthreads();
  for (int e = tid; e < a.n_rows; e += TH) {
    float s = 0.f;
    for (int i = 0; i < TH / 64; ++i) s += part[i][e];
    a.rows_out[(size_t)t * a.n_rows + e] = s;
  }
}

// NV: pieces of four columns a thread, TH threads
template <int S, int NV, int TH>
__global__ __launch_bounds__(TH) void hyper_step_kernel(HyperArgs a) {
  __shared__ float red[20];
  __shared__ float part[TH / 64][MAX_ROWS];
  const int t = blockIdx.x, tid = threadIdx.x, D = a.D;
  float mix[S][S], wo[S], wi[S];
#pragma unroll
  for (int s = 0; s < S; ++s) {
    wi[s] = a.in ? a.in[s] : 1.f;
    wo[s] = a.y ? a.out[s] : 0.f;
#pragma unroll
    for (int r = 0; r < S; ++r) mix[s][r] = a.y ? a.mix[s * S + r] : 0.f;
  }
  f32x4_t u[NV];
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = 4 * (tid + TH * i);
    u[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (c >= D) continue;
    f32x4_t x[S];
    if (a.xs) {
#pragma unroll
      for (int s = 0; s < S; ++s) x[s] = *(const f32x4_t*)(a.xs + ((size_t)t * S + s) * D + c);
    } else {
      const f32x4_t f = *(const f32x4_t*)(a.first + (size_t)t * a.ld_first + c);
#pragma unroll
      for (int s = 0; s < S; ++s) x[s] = f;
    }
    if (a.y) {
      f32x4_t y = a.bias ? *(const f32x4_t*)(a.bias + c) : f32x4_t{0.f, 0.f, 0.f, 0.f};
      const float* yp = a.y + (size_t)t * a.ldy + c;
      int p = 0;
      for (; p + 4 <= a.n_parts; p += 4) {
        const f32x4_t y0 = *(const f32x4_t*)(yp + p * a.y_part), y1 = *(const f32x4_t*)(yp + (p + 1) * a.y_part);
        const f32x4_t y2 = *(const f32x4_t*)(yp + (p + 2) * a.y_part), y3 = *(const f32x4_t*)(yp + (p + 3) * a.y_part);
        y += y0, y += y1, y += y2, y += y3;
      }
      for (; p < a.n_parts; ++p) y += *(const f32x4_t*)(yp + p * a.y_part);
      f32x4_t n[S];
#pragma unroll
      for (int r = 0; r < S; ++r) {
        n[r] = mix[0][r] * x[0];
#pragma unroll
        for (int s = 1; s < S; ++s) n[r] += mix[s][r] * x[s];
        n[r] += wo[r] * y;
      }
#pragma unroll
      for (int s = 0; s < S; ++s) x[s] = n[s];
    }
    if (a.xs_out) {
#pragma unroll
      for (int s = 0; s < S; ++s) *(f32x4_t*)(a.xs_out + ((size_t)t * S + s) * D + c) = x[s];
    }
    f32x4_t v = wi[0] * x[0];
#pragma unroll
    for (int s = 1; s < S; ++s) v += wi[s] * x[s];
    u[i] = v;
    sum += (v[0] + v[1]) + (v[2] + v[3]);
    if (a.sum_out) *(f32x4_t*)(a.sum_out + (size_t)t * a.ld_sum + c) = v;
  }
  if (!a.norm_out) return;  // (the whole block)
  const float mean = block_sum(sum, red) / (float)D;
  float sq = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    if (4 * (tid + TH * i) >= D) continue;
    u[i] -= mean;
    sq += (u[i][0] * u[i][0] + u[i][1] * u[i][1]) + (u[i][2] * u[i][2] + u[i][3] * u[i][3]);
  }
  const float rstd = 1.0f / sqrtf(block_sum(sq, red) / (float)D + a.eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = 4 * (tid + TH * i);
    if (c >= D) continue;
    f32x4_t v = u[i] * rstd;
    if (a.gamma) v *= *(const f32x4_t*)(a.gamma + c);
    if (a.beta) v += *(const f32x4_t*)(a.beta + c);
    if (a.norm_dtype == DT_BF16) {
      const uint2 b = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
      *(uint2*)((bf16*)a.norm_out + (size_t)t * D + c) = b;
      u[i] = four((const bf16*)&b);  // (the product takes the row as it is written)
    } else {
      *(f32x4_t*)((float*)a.norm_out + (size_t)t * D + c) = v;
      u[i] = v;
    }
  }
  if (!a.w) return;
  if (a.norm_dtype == DT_BF16) small_rows<bf16, NV, TH>(a, t, u, part);
  else small_rows<float, NV, TH>(a, t, u, part);
}

DEFINE_LAST_ERROR(mlxlm_last_error)

template <int S>
static void launch(const HyperArgs& a, hipStream_t stream) {
#define RUN(NV, TH) hipLaunchKernelGGL((hyper_step_kernel<S, NV, TH>), dim3(a.T), dim3(TH), 0, stream, a)
  if (a.D <= 1024) RUN(1, 256);
  else if (a.D <= 2048) RUN(2, 256);
  else if (a.D <= 4096) RUN(4, 256);
  else if (a.D <= 8192) RUN(2, 1024);
  else RUN(8, 1024);
#undef RUN
}

extern "C" int hyper_step(const HyperArgs* args, hipStream_t stream) {
  const HyperArgs& a = *args;
  if (a.T <= 0) return 0;
  if (a.D <= 0 || a.D % 4 || a.D > 32768) FAIL("hyper_step: rows of %d columns (a multiple of 4, at most 32768)", a.D);
  if (a.S < 1 || a.S > MAX_STREAMS) FAIL("hyper_step: %d streams (1 to %d)", a.S, MAX_STREAMS);
  if ((!a.xs && !a.first) || (!a.norm_out && !a.sum_out && !a.xs_out)) FAIL("hyper_step: nothing to read, or nothing to write");
  if (!a.xs && (a.ld_first < a.D || a.ld_first % 4)) FAIL("hyper_step: the first rows' stride %d", a.ld_first);
  if (a.y && (!a.mix || !a.out || a.n_parts < 1 || a.ldy < a.D || a.ldy % 4 || a.y_part % 4)) FAIL("hyper_step: a write needs its weights and whole rows");
  if (a.sum_out && (a.ld_sum < a.D || a.ld_sum % 4)) FAIL("hyper_step: the sum's row stride %d", a.ld_sum);
  if (a.norm_out && a.norm_dtype != DT_F32 && a.norm_dtype != DT_BF16) FAIL("hyper_step: unknown dtype code %d", a.norm_dtype);
  if (a.w && (!a.norm_out || !a.rows_out || a.n_rows <= 0 || a.n_rows > MAX_ROWS || ((uintptr_t)a.w & 15)))
    FAIL("hyper_step: a product of %d rows (1 to %d) with the norm", a.n_rows, MAX_ROWS);
  if (((uintptr_t)a.xs | (uintptr_t)a.first | (uintptr_t)a.xs_out | (uintptr_t)a.y | (uintptr_t)a.norm_out | (uintptr_t)a.sum_out |
       (uintptr_t)a.gamma | (uintptr_t)a.beta | (uintptr_t)a.bias) & 15)
    FAIL("hyper_step: 16-byte aligned rows");
  switch (a.S) {
    case 1: launch<1>(a, stream); break;
    case 2: launch<2>(a, stream); break;
    case 3: launch<3>(a, stream); break;
    case 4: launch<4>(a, stream); break;
    case 5: launch<5>(a, stream); break;
    case 6: launch<6>(a, stream); break;
    case 7: launch<7>(a, stream); break;
    default: launch<8>(a, stream); break;
  }
  CHECK_LAUNCH("hyper_step");
  return 0;
}
