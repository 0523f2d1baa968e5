// The real-gated linear recurrent unit with its short convolution, over W channels in B equal parts:
//   u = conv(x) + bias (per channel, `taps` inputs, zeros before the start)
//   r = sigmoid(Ra[b] u_b + ra.b),  i = sigmoid(Ri[b] u_b + ri.b)        (a square matrix a part)
//   log a = -8 r softplus(lam),  a = exp(log a)
//   S_t = a S_(t-1) + sqrt(1 - a^2) i u,   out = S * gelu_tanh(y)
// x and y are float columns of a projection's rows.  The convolution's last inputs lie in the request's
// state row as a ring, position p in row p % taps: a step's rows are none of those it still reads, so
// blocks that need the same inputs run side by side.
//
//   rglru_gates  portions: a block a (64 tokens of a request, 64 channels of a part): the convolution into LDS, both gates on
//                the matrix cores, a and sqrt(1 - a^2) i u as rows, and what the 64 tokens do to the
//                state (S -> A S + B a channel), each lane's tokens composed, then lanes, then waves
//   rglru_scan   a thread a channel of 64 tokens: the state ahead of them from the A, B of the request's
//                earlier ones, then token by token, the output's gate on the way out; the request's
//                last one leaves the state and the ring
//   rglru_step   one token a request: a block sixteen channels of a part for up to sixteen requests, all
//                of the above in one launch
//
// All 32-bit but `out` (the gates' products: rows_product.h).
#include "common.h"
#include "rows_product.h"

#define LOG2E 1.4426950408889634f
// (on the hardware's exponential and reciprocal, an ulp or two each)
__device__ __forceinline__ float exp_f(float x) { return __builtin_amdgcn_exp2f(x * LOG2E); }
__device__ __forceinline__ float sigmoid_f(float z) { return __builtin_amdgcn_rcpf(1.0f + exp_f(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

#define SPAN 64

struct RglruArgs {
  const float* x;  // [rows, ldx]: W columns that the convolution reads
  const float* y;  // [rows, ldx]: W columns of the output's gate, ahead of its gelu
  int ldx;
  const float* conv_w;  // [W][taps]
  const float* conv_b;  // [W] or null
  int taps;
  const void* ra;  // [B][w][wp], columns from w on zero
  const void* ri;
  const float* ra_b;  // [W]
  const float* ri_b;
  const float* lam;  // [W]
  float* state;      // a request's row: W floats of S at state_offset, the ring [taps][W] at ring_offset
  size_t state_stride, state_offset, ring_offset;
  const int* positions;
  const int* seq_start;
  const int* seq_len;
  const int* slot_ids;
  const int* span_req;    // portions: [spans]
  const int* span_start;  // first token, counted from the request's first of this step
  const int* span_first;  // [requests]
  float* a;        // [rows, W]
  float* b;        // [rows, W]
  float2* does;    // [spans, W]
  float* s0;       // [requests, W] the state ahead of the step
  void* out;       // [rows, ldo]
  int ldo, dtype;  // of the weights and of out
  int n_requests, n_spans, W, B, w, wp;
  float decay;  // the 8 of log a
};

// The convolution's output for channel c of the token at flat row `row`, `local` tokens into its portion.
__device__ __forceinline__ float conv_at(const RglruArgs& p, const float* ring, int row, int local, int pos, int c) {
  const float* w = p.conv_w + (size_t)c * p.taps;
  float acc = 0.f;
  for (int j = p.taps - 1; j >= 0; --j) {  // the oldest input first
    float in = 0.f;
    if (local - j >= 0)
      in = p.x[(size_t)(row - j) * p.ldx + c];
    else if (pos - j >= 0)
      in = ring[(size_t)((pos - j) % p.taps) * p.W + c];
    acc += w[p.taps - 1 - j] * in;
  }
  return acc + (p.conv_b ? p.conv_b[c] : 0.f);
}

// The same for CONV_TILE tokens in a row of one channel, all inputs asked for at once (up to CONV_TAPS
// taps).  `live` of the tokens exist; at or below -CONV_TAPS nothing is read.
#define CONV_TAPS 8
#define CONV_TILE 8
__device__ __forceinline__ void conv_run(const RglruArgs& p, const float* ring, int row, int local, int pos, int live, int c, float* out, int ld) {
  float w[CONV_TAPS], in[CONV_TILE + CONV_TAPS - 1];
#pragma unroll
  for (int j = 0; j < CONV_TAPS; ++j) w[j] = j < p.taps ? p.conv_w[(size_t)c * p.taps + p.taps - 1 - j] : 0.f;  // (of the input j tokens back)
  if (local >= CONV_TAPS - 1 && live >= 1) {  // all of them in the step's own rows
    const float* x = p.x + (size_t)(row - (CONV_TAPS - 1)) * p.ldx + c;
    const int last = live - 1 + CONV_TAPS - 1;
#pragma unroll
    for (int i = 0; i < CONV_TILE + CONV_TAPS - 1; ++i) in[i] = x[(size_t)min(i, last) * p.ldx];  // (beyond the last: not used)
  } else {
#pragma unroll
    for (int i = 0; i < CONV_TILE + CONV_TAPS - 1; ++i) {
      const int d = i - (CONV_TAPS - 1);  // tokens from the first of the run
      in[i] = 0.f;
      if (d >= live || -d >= p.taps) continue;
      if (local + d >= 0) in[i] = p.x[(size_t)(row + d) * p.ldx + c];
      else if (pos + d >= 0) in[i] = ring[(size_t)((pos + d) % p.taps) * p.W + c];
    }
  }
  const float shift = p.conv_b ? p.conv_b[c] : 0.f;
#pragma unroll
  for (int t = 0; t < CONV_TILE; ++t) {
    float acc = 0.f;
#pragma unroll
    for (int j = CONV_TAPS - 1; j >= 0; --j) acc += w[j] * in[t + CONV_TAPS - 1 - j];  // the oldest input first
    out[t * ld] = t < live ? acc + shift : 0.f;
  }
}

struct Gated {
  float a, b;
};
__device__ __forceinline__ Gated gated(float zr, float zi, float u, float rate) {
  const float log_a = -rate * sigmoid_f(zr), a = exp_f(log_a), t = 2.0f * log_a;
  // 1 - a^2 = -(exp(t) - 1): near t = 0 as a series, without cancellation
  const float series = -t * (1.0f + t * (0.5f + t * (1.0f / 6 + t * (1.0f / 24 + t * (1.0f / 120 + t * (1.0f / 720))))));
  return Gated{a, sqrtf(t > -0.25f ? series : 1.0f - a * a) * sigmoid_f(zi) * u};
}

// TT: tokens in LDS at a time (64, or 16 for wide parts); TH threads: TT / 16 tiles of rows, the waves'
// remaining factor over the block's 64 channels (every block makes the whole part's convolution).
template <typename T, int TT, int TH>
__global__ __launch_bounds__(TH) void rglru_gates_kernel(RglruArgs p) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float2 does[4][64];
  constexpr int RT = TT / 16, CW = TH / 64 / RT, NJ = 4 / CW;  // NJ: tiles of sixteen channels a wave
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lr = lane & 15, lg = lane >> 4;
  const int rt = wave % RT, j0 = wave / RT * NJ;
  const int w = p.w, wp = p.wp, ld = wp + 4;
  float* U = lds;  // [TT][ld]
  const int slices = (w + 63) / 64, span = blockIdx.x, part = blockIdx.y / slices, s0 = blockIdx.y % slices * 64, c0 = part * w;
  const int r = p.span_req[span], lo = p.span_start[span], n = min(SPAN, p.seq_len[r] - lo);
  const int row0 = p.seq_start[r] + lo, pos0 = p.positions[row0];
  const float* srow = p.state + (size_t)p.slot_ids[r] * p.state_stride;
  const float* ring = srow + p.ring_offset;
  if (lo == 0 && tid < 64 && s0 + tid < w) p.s0[(size_t)r * p.W + c0 + s0 + tid] = srow[p.state_offset + c0 + s0 + tid];
  const T* gate[2 * NJ];
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    const size_t f = (size_t)(part * w + min(s0 + 16 * (j0 + j) + lr, w - 1)) * wp;
    gate[j] = (const T*)p.ra + f, gate[NJ + j] = (const T*)p.ri + f;
  }
  const bool run = p.taps <= CONV_TAPS;
  for (int t0 = 0; t0 < n; t0 += TT) {
    if (t0 > 0) __syncthreads();  // the tile before is done with U
    if (run) {
      for (int e = tid; e < TT / CONV_TILE * wp; e += TH) {
        const int t = e / wp * CONV_TILE, c = e % wp, first = t0 + t;
        conv_run(p, ring, row0 + first, lo + first, pos0 + first, c < w ? n - first : -CONV_TAPS, c0 + min(c, w - 1), U + t * ld + c, ld);
      }
    } else {
      for (int e = tid; e < TT * wp; e += TH) {
        const int t = e / wp, c = e - t * wp;
        U[t * ld + c] = c < w && t0 + t < n ? conv_at(p, ring, row0 + t0 + t, lo + t0 + t, pos0 + t0 + t, c0 + c) : 0.f;
      }
    }
    __syncthreads();
    const float* urow = U + (16 * rt + lr) * ld;
    f32x4_t z[2 * NJ];
#pragma unroll
    for (int j = 0; j < 2 * NJ; ++j) z[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    rows_product<2 * NJ>([&](int k) { return *(const float4*)(urow + k); }, gate, wp, 0, 1, z);
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      const int sc = 16 * (j0 + j) + lr, cc = s0 + sc;
      const bool live = cc < w;
      const int c = c0 + min(cc, w - 1);
      const float rb = p.ra_b[c], ib = p.ri_b[c], rate = p.decay * softplus_f(p.lam[c]);
      float A = 1.f, Bv = 0.f;
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const int t = 16 * rt + 4 * lg + x;
        if (t0 + t < n && live) {
          const Gated g = gated(z[j][x] + rb, z[NJ + j][x] + ib, U[t * ld + cc], rate);
          const size_t at = (size_t)(row0 + t0 + t) * p.W + c;
          p.a[at] = g.a, p.b[at] = g.b;
          Bv = g.a * Bv + g.b, A *= g.a;
        }
      }
      // lanes of the same channel, sixteen apart, hold four tokens each, in order
#pragma unroll
      for (int step = 16; step < 64; step *= 2) {
        const float A2 = __shfl_xor(A, step, 64), B2 = __shfl_xor(Bv, step, 64);
        const bool later = lane & step;
        Bv = later ? A * B2 + Bv : A2 * Bv + B2;
        A *= A2;
      }
      if (lg == 0) {
        float2* at = &does[rt][sc];
        if (TT < SPAN && t0 > 0)
          *at = make_float2(at->x * A, A * at->y + Bv);  // (RT == 1: this tile's tokens follow the last one's)
        else
          *at = make_float2(A, Bv);
      }
    }
  }
  __syncthreads();
  if (tid < 64 && s0 + tid < w) {
    float A = 1.f, Bv = 0.f;
#pragma unroll
    for (int i = 0; i < RT; ++i) {
      const float2 d = does[i][tid];
      Bv = d.x * Bv + d.y, A *= d.x;
    }
    p.does[(size_t)span * p.W + c0 + s0 + tid] = make_float2(A, Bv);
  }
}

// Block (span, 256 channels).
template <typename T>
__global__ __launch_bounds__(256) void rglru_scan_kernel(RglruArgs p) {
  const int c = blockIdx.y * 256 + threadIdx.x, span = blockIdx.x;
  if (c >= p.W) return;  // (no barrier follows)
  const int r = p.span_req[span], lo = p.span_start[span], len = p.seq_len[r], n = min(SPAN, len - lo);
  const int row0 = p.seq_start[r] + lo;
  float S = p.s0[(size_t)r * p.W + c];
  const int first = p.span_first[r];
  for (int s = first; s < span; s += 8) {
    float2 d[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) d[i] = p.does[(size_t)min(s + i, span - 1) * p.W + c];
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (s + i < span) S = d[i].x * S + d[i].y;
  }
  for (int t = 0; t < n; t += 16) {
    float a[16], b[16], y[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const size_t row = (size_t)(row0 + min(t + i, n - 1));
      a[i] = p.a[row * p.W + c], b[i] = p.b[row * p.W + c], y[i] = p.y[row * p.ldx + c];
    }
#pragma unroll
    for (int i = 0; i < 16; ++i)
      if (t + i < n) {
        S = a[i] * S + b[i];
        ((T*)p.out)[(size_t)(row0 + t + i) * p.ldo + c] = from_f32<T>(S * gelu_tanh(y[i]));
      }
  }
  if (lo + n == len) {  // the request's last tokens of this step
    float* srow = p.state + (size_t)p.slot_ids[r] * p.state_stride;
    srow[p.state_offset + c] = S;
    if (p.taps > 1) {
      const int start = p.seq_start[r], pos = p.positions[start];
      for (int t = max(0, len - (p.taps - 1)); t < len; ++t)
        srow[p.ring_offset + (size_t)((pos + t) % p.taps) * p.W + c] = p.x[(size_t)(start + t) * p.ldx + c];
    }
  }
}

// The two gates' weights that a wave of rglru_step takes first, asked for before the rows are there (bfloat16).
template <typename T>
struct Ahead {
  __device__ __forceinline__ void ask(const T* const (&)[2], int, int) {}
  template <typename Rows>
  __device__ __forceinline__ void product(Rows x, const T* const (&w)[2], int K, int wave, f32x4_t (&z)[2]) {
    rows_product<2>(x, w, K, wave, 4, z);
  }
};
template <>
struct Ahead<bf16> {
  PiecesAhead<2, 2> pieces;
  __device__ __forceinline__ void ask(const bf16* const (&w)[2], int K, int wave) { pieces.ask(w, K, wave, 4); }
  template <typename Rows>
  __device__ __forceinline__ void product(Rows x, const bf16* const (&w)[2], int K, int wave, f32x4_t (&z)[2]) {
    pieces.product(x, K, wave, 4, z);
    rows_product<2>(x, w, K, wave + 4 * 2, 4, z);
  }
};

// Block (part x 16 channels, 16 requests of one token each): four waves share K, a thread then a (request, channel).
template <typename T>
__global__ __launch_bounds__(256) void rglru_step_kernel(RglruArgs p) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float part[2][4][16][17];
  __shared__ int s_row[16], s_pos[16], s_place[16][CONV_TAPS];  // place: where in the ring the input j tokens back lies
  __shared__ const float* s_ring[16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lr = lane & 15, lg = lane >> 4;
  const int w = p.w, wp = p.wp, ld = wp + 4, tiles = (w + 15) / 16;
  const int b = blockIdx.x / tiles, f0 = 16 * (blockIdx.x % tiles), c0 = b * w;
  const int r0 = blockIdx.y * 16, n = min(16, p.n_requests - r0);
  float* U = lds;  // [16][ld]
  // what the end of the block reads, asked for first
  const int er = tid >> 4, ec = f0 + (tid & 15);
  const bool mine = er < n && ec < w;
  const int req = r0 + min(er, n - 1), c = c0 + min(ec, w - 1), erow = p.seq_start[req];
  float* srow = p.state + (size_t)p.slot_ids[req] * p.state_stride;
  const float S = srow[p.state_offset + c], y = p.y[(size_t)erow * p.ldx + c], x = p.x[(size_t)erow * p.ldx + c];
  const float rb = p.ra_b[c], ib = p.ri_b[c], lam = p.lam[c];
  const size_t f = (size_t)(b * w + min(f0 + lr, w - 1)) * wp;
  const T* const gates[2] = {(const T*)p.ra + f, (const T*)p.ri + f};
  const bool run = p.taps <= CONV_TAPS;
  Ahead<T> ahead;
  ahead.ask(gates, wp, wave);
  if (tid < 16 * CONV_TAPS) {
    const int t = tid / CONV_TAPS, j = tid % CONV_TAPS;
    if (t < n) {
      const int row = p.seq_start[r0 + t], pos = p.positions[row];
      s_place[t][j] = j < p.taps ? (pos + p.taps - j) % p.taps : 0;
      if (j == 0) s_row[t] = row, s_pos[t] = pos, s_ring[t] = p.state + (size_t)p.slot_ids[r0 + t] * p.state_stride + p.ring_offset;
    }
  }
  __syncthreads();
#pragma unroll 2
  for (int e = tid; e < n * wp; e += 256) {
    const int t = e / wp, k = e - t * wp, row = s_row[t], pos = s_pos[t];
    const float* ring = s_ring[t];
    const int ch = c0 + min(k, w - 1);
    float u;
    if (run) {  // all inputs asked for at once
      float in[CONV_TAPS], cw[CONV_TAPS];
#pragma unroll
      for (int j = 0; j < CONV_TAPS; ++j) {
        in[j] = cw[j] = 0.f;
        if (j >= p.taps) continue;
        cw[j] = p.conv_w[(size_t)ch * p.taps + p.taps - 1 - j];
        in[j] = j == 0 ? p.x[(size_t)row * p.ldx + ch] : ring[(size_t)s_place[t][j] * p.W + ch];
      }
      u = p.conv_b ? p.conv_b[ch] : 0.f;
      float acc = 0.f;
#pragma unroll
      for (int j = CONV_TAPS - 1; j >= 0; --j) acc += pos - j >= 0 ? cw[j] * in[j] : 0.f;
      u += acc;
    } else {
      u = conv_at(p, ring, row, 0, pos, ch);
    }
    U[t * ld + k] = k < w ? u : 0.f;
  }
  for (int e = n * ld + tid; e < 16 * ld; e += 256) U[e] = 0.f;
  __syncthreads();
  const float* urow = U + lr * ld;
  auto row = [&](int k) { return *(const float4*)(urow + k); };
  f32x4_t z[2] = {f32x4_t{0.f, 0.f, 0.f, 0.f}, f32x4_t{0.f, 0.f, 0.f, 0.f}};
  ahead.product(row, gates, wp, wave, z);
#pragma unroll
  for (int i = 0; i < 4; ++i) part[0][wave][4 * lg + i][lr] = z[0][i], part[1][wave][4 * lg + i][lr] = z[1][i];
  __syncthreads();
  if (!mine) return;
  const int q = tid & 15;
  const float zr = ((part[0][0][er][q] + part[0][1][er][q]) + (part[0][2][er][q] + part[0][3][er][q])) + rb;
  const float zi = ((part[1][0][er][q] + part[1][1][er][q]) + (part[1][2][er][q] + part[1][3][er][q])) + ib;
  const Gated g = gated(zr, zi, U[er * ld + ec], p.decay * softplus_f(lam));
  const float Sn = g.a * S + g.b;
  srow[p.state_offset + c] = Sn;
  if (p.taps > 1) srow[p.ring_offset + (size_t)(p.positions[erow] % p.taps) * p.W + c] = x;
  ((T*)p.out)[(size_t)erow * p.ldo + c] = from_f32<T>(Sn * gelu_tanh(y));
}

DEFINE_LAST_ERROR(mlxlm_last_error)

#define LDS_MOST (150 * 1024)
static size_t gates_lds(int tt, int w, int wp) {
  (void)w;
  return (size_t)tt * (wp + 4) * sizeof(float);
}

// 1 if the kernels take parts of w channels
extern "C" int rglru_takes(int w) {
  const int wp = (w + 7) / 8 * 8;
  return w > 0 && gates_lds(16, w, wp) <= LDS_MOST;
}

static int check(const RglruArgs& a, const char* who) {
  if (!a.x || !a.y || !a.conv_w || !a.ra || !a.ri || !a.ra_b || !a.ri_b || !a.lam || !a.state || !a.positions || !a.seq_start ||
      !a.seq_len || !a.slot_ids || !a.out)
    FAIL("%s: null pointer", who);
  if (a.B <= 0 || a.w <= 0 || a.W != a.B * a.w || a.wp % 8 || a.wp < a.w || !rglru_takes(a.w)) FAIL("%s: %d parts of %d channels", who, a.B, a.w);
  if (a.taps < 1 || a.ldx < a.W || a.ldo < a.W) FAIL("%s: %d taps, rows of %d and %d for %d channels", who, a.taps, a.ldx, a.ldo, a.W);
  if (a.state_stride < a.state_offset + a.W || (a.taps > 1 && a.state_stride < a.ring_offset + (size_t)a.taps * a.W))
    FAIL("%s: the state rows are too short", who);
  if (!(a.decay > 0.f)) FAIL("%s: the decay's constant %g", who, (double)a.decay);
  if (((uintptr_t)a.ra | (uintptr_t)a.ri) & 15) FAIL("%s: 16-byte aligned weights", who);
  if (a.dtype != DT_F32 && a.dtype != DT_BF16) FAIL("%s: unknown dtype code %d", who, a.dtype);
  return 0;
}

template <typename K>
static void allow(K kernel) {
  (void)hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, LDS_MOST);
}

extern "C" int rglru_step(const RglruArgs* args, hipStream_t stream) {
  const RglruArgs& a = *args;
  if (a.n_requests <= 0) return 0;
  if (check(a, "rglru_step")) return 1;
  const dim3 grid(a.B * ((a.w + 15) / 16), (a.n_requests + 15) / 16), block(256);
  const size_t lds = (size_t)16 * (a.wp + 4) * sizeof(float);
  static bool raised = false;
  if (!raised) allow(rglru_step_kernel<float>), allow(rglru_step_kernel<bf16>), raised = true;
  if (a.dtype == DT_F32) hipLaunchKernelGGL(rglru_step_kernel<float>, grid, block, lds, stream, a);
  else hipLaunchKernelGGL(rglru_step_kernel<bf16>, grid, block, lds, stream, a);
  CHECK_LAUNCH("rglru_step");
  return 0;
}

extern "C" int rglru_portions(const RglruArgs* args, hipStream_t stream) {
  const RglruArgs& a = *args;
  if (a.n_requests <= 0 || a.n_spans <= 0) return 0;
  if (check(a, "rglru_portions")) return 1;
  if (!a.span_req || !a.span_start || !a.span_first || !a.a || !a.b || !a.does || !a.s0) FAIL("rglru_portions: null pointer");
  static bool raised = false;
  if (!raised) {
    allow(rglru_gates_kernel<float, 64, 1024>), allow(rglru_gates_kernel<float, 16, 256>);
    allow(rglru_gates_kernel<bf16, 64, 1024>), allow(rglru_gates_kernel<bf16, 16, 256>);
    raised = true;
  }
  const bool wide = gates_lds(64, a.w, a.wp) > 80 * 1024;  // (two blocks a CU)
  const dim3 grid(a.n_spans, a.B * ((a.w + 63) / 64)), scan(a.n_spans, (a.W + 255) / 256), block(256), wide_block(1024);
  const size_t lds = gates_lds(wide ? 16 : 64, a.w, a.wp);
  if (a.dtype == DT_F32) {
    if (wide) hipLaunchKernelGGL((rglru_gates_kernel<float, 16, 256>), grid, block, lds, stream, a);
    else hipLaunchKernelGGL((rglru_gates_kernel<float, 64, 1024>), grid, wide_block, lds, stream, a);
    hipLaunchKernelGGL(rglru_scan_kernel<float>, scan, block, 0, stream, a);
  } else {
    if (wide) hipLaunchKernelGGL((rglru_gates_kernel<bf16, 16, 256>), grid, block, lds, stream, a);
    else hipLaunchKernelGGL((rglru_gates_kernel<bf16, 64, 1024>), grid, wide_block, lds, stream, a);
    hipLaunchKernelGGL(rglru_scan_kernel<bf16>, scan, block, 0, stream, a);
  }
  CHECK_LAUNCH("rglru_portions");
  return 0;
}
