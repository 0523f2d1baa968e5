// The gated delta rule for portions of many tokens:
//   S_t = g_t S_(t-1) + k_t u_t^T,   u_t = beta_t (v_t - g_t S_(t-1)^T k_t),   o_t = S_t^T q_t
// (k_t of unit length, S [N][P] per request and head, 32-bit), in chunks of 64 tokens.  With L_t the
// sum of log g inside the chunk and A[t][j] = beta_t exp(L_t - L_j) (k_t . k_j) for j < t, else 0,
//   (1 + A) U = diag(beta) (V - diag(exp L) K S_0)
//   O   = diag(exp L) Q S_0 + tril(exp(L_t - L_j) q_t . k_j) U
//   S_C = exp(L_C) S_0 + sum_j exp(L_C - L_j) k_j u_j^T
// so what a chunk does to the state is one lower triangular system and a few small products, and only
// S_0 of a chunk waits for the chunk before it:
//
//   delta_prepare  the projection's columns to the recurrence's operands, a wave a head of a row:
//                  causal convolution per channel and silu, queries and keys to unit vectors (queries
//                  scaled), beta = sigmoid(.), log g = -exp(A_log) softplus(. + dt_bias).  Heads are
//                  padded with zeros to multiples of sixteen columns.  The convolution's last inputs
//                  lie in the request's state row as a ring (position p in row p % taps); the waves
//                  of a request's first row take all rows that read it, then write it.
//   delta_solve    a block a (head, chunk): A, (1 + A)^-1 (by blocks of sixteen), and with it
//                  W = (1 + A)^-1 diag(beta exp L) K and U_0 = (1 + A)^-1 diag(beta) V: U = U_0 - W S_0.
//   delta_states   a block a (head, request, sixteen value columns), chunk after chunk: U in place of
//                  U_0, the state ahead of every chunk, the request's new state.  The state's columns
//                  do not meet, so they are dealt to blocks; S stays in registers.
//   delta_outputs  a block a (head, chunk): O, divided by its root mean square, times a weight and
//                  silu(gate) (or sigmoid(gate)).
//
// With a decay per key channel L_t is a vector over the key columns, and what was a number between two
// scalar products goes inside: A[t][j] = beta_t sum_n k_t[n] k_j[n] exp(L_t[n] - L_j[n]), likewise q_t . k_j.
// For the matrix cores the exponent is cut in two at a reference R[n] that lies between the tokens:
// (k_t exp(L_t - R)) . (k_j exp(R - L_j)).  For two tiles of sixteen tokens R is L ahead of the later
// tile, so both exponents are at most 0; within a tile R is L at its middle, which is safe while L falls
// by less than FAR_APART on either side of it, and a tile with a faster channel is summed pair by pair.
//   lowrank_gates  log g and the output gate's logits from their narrow middles (rows_product.h)
//   delta_solve_channel  in place of delta_solve; it leaves everything that the exponents enter for the
//                  others: q_t . k_j with the decays between, exp(L_t) q_t, exp(L_C - L_j) k_j, exp(L_C)
//
// All 32-bit, the products on v_mfma_f32_16x16x4_f32 (lane l brings A[l % 16][l / 16] and
// B[l / 16][l % 16] and gets D[4 (l / 16) + x][l % 16]; where both operands run over the same
// columns, a lane brings four consecutive ones to four instructions).
#include "common.h"
#include "rows_product.h"

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

#define UNIT_EPS 1e-6f  // a unit vector is x / sqrt(sum(x^2) + UNIT_EPS)
#define C 64            // tokens a chunk
#define CS 68           // row stride of the chunk's square arrays
#define SS 20           // row stride of sixteen columns of the state
#define MAX_N 256       // key columns (padded) that delta_states holds in registers
#define MAX_P 256
#define PREPARE_MAX 512  // the widest head that delta_prepare takes

#define MFMA(a, b, c) __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0)

struct DeltaPrepareArgs {
  const float* u;  // [rows, ldu]: q (Hk heads of N), k (Hk of N), v (H of P) from column 0 on
  int ldu, b_col, a_col;
  int n_rows, H, Hk, N, P;
  const float* conv_w;  // [channels][taps]
  int taps;
  const float* A_log;
  const float* dt_bias;
  float q_scale;
  float* state;  // the ring: [taps][channels] at ring_offset of a request's row
  size_t state_stride, ring_offset;
  const int* token_req;
  const int* positions;
  const int* seq_start;
  const int* seq_len;
  const int* slot_ids;
  float* q;  // [rows, Hk * Np]
  float* k;
  float* v;  // [rows, H * Pp]
  float* log_g;  // [rows, H], or null: made elsewhere (a decay per key channel)
  float* beta;
};

__global__ __launch_bounds__(256) void delta_prepare_kernel(DeltaPrepareArgs a) {
  const int row0 = blockIdx.x, lane = threadIdx.x & 63, item = blockIdx.y * 4 + (threadIdx.x >> 6);
  const int Np = (a.N + 15) & ~15, Pp = (a.P + 15) & ~15;
  if (item > 2 * a.Hk + a.H) return;  // whole waves leave; no barrier follows
  if (item == 2 * a.Hk + a.H) {
    const float* ur = a.u + (size_t)row0 * a.ldu;
    for (int h = lane; h < a.H; h += 64) {
      a.beta[(size_t)row0 * a.H + h] = 1.0f / (1.0f + expf(-ur[a.b_col + h]));
      if (a.log_g) a.log_g[(size_t)row0 * a.H + h] = -expf(a.A_log[h]) * softplus_f(ur[a.a_col + h] + a.dt_bias[h]);
    }
    return;
  }
  const int req = a.token_req[row0], start = a.seq_start[req], n = a.seq_len[req], local0 = row0 - start;
  if (local0 > 0 && local0 < a.taps - 1) return;  // (its request's first row's waves take this row too)
  const int kind = item < a.Hk ? 0 : item < 2 * a.Hk ? 1 : 2, hd = item - (kind == 0 ? 0 : kind == 1 ? a.Hk : 2 * a.Hk);
  const int dim = kind == 2 ? a.P : a.N, padded = kind == 2 ? Pp : Np, heads = kind == 2 ? a.H : a.Hk;
  const int ch0 = kind == 0 ? hd * a.N : kind == 1 ? a.Hk * a.N + hd * a.N : 2 * a.Hk * a.N + hd * a.P;
  const int channels = 2 * a.Hk * a.N + a.H * a.P;
  float* dst = (kind == 0 ? a.q : kind == 1 ? a.k : a.v) + hd * padded;
  float* ring = a.state + (size_t)a.slot_ids[req] * a.state_stride + a.ring_offset;
  const int rows = local0 == 0 ? max(1, min(n, a.taps - 1)) : 1;
  for (int rr = 0; rr < rows; ++rr) {
    const int row = row0 + rr, local = local0 + rr, pos = a.positions[row];
    float y[PREPARE_MAX / 64], ss = 0.f;
#pragma unroll
    for (int i = 0; i < PREPARE_MAX / 64; ++i) {
      const int c = lane + 64 * i;
      y[i] = 0.f;
      if (c < dim) {
        const int ch = ch0 + c;
        const float* w = a.conv_w + (size_t)ch * a.taps;
        float acc = 0.f;
        for (int j = a.taps - 1; j >= 0; --j) {  // the oldest input first
          float in = 0.f;
          if (local - j >= 0)
            in = a.u[(size_t)(row - j) * a.ldu + ch];
          else if (pos - j >= 0)
            in = ring[(size_t)((pos - j) % a.taps) * channels + ch];
          acc += w[a.taps - 1 - j] * in;
        }
        y[i] = silu_f(acc);
        ss += y[i] * y[i];
      }
    }
    const float f = kind == 2 ? 1.f : (kind == 0 ? a.q_scale : 1.f) / sqrtf(wave_sum(ss) + UNIT_EPS);
#pragma unroll
    for (int i = 0; i < PREPARE_MAX / 64; ++i) {
      const int c = lane + 64 * i;
      if (c < padded) dst[(size_t)row * heads * padded + c] = y[i] * f;
    }
  }
  if (local0 == 0 && a.taps > 1) {
    const int pos0 = a.positions[row0];
    for (int t = max(0, n - (a.taps - 1)); t < n; ++t)
      for (int c = lane; c < dim; c += 64)
        ring[(size_t)((pos0 + t) % a.taps) * channels + ch0 + c] = a.u[(size_t)(start + t) * a.ldu + ch0 + c];
  }
}

struct DeltaChunkArgs {
  const float* q;  // [rows, Hk * Np]
  const float* k;
  const float* v;      // [rows, H * Pp]
  const float* log_g;  // [rows, H]; by channel [rows, H * Np]
  const float* beta;
  float* cum;        // [rows, H] L inside the chunk
  float* w;          // [rows, H * Np]
  float* u;          // [rows, H * Pp] U_0, then U
  float* states;     // [chunks, H, Np, Pp] the state ahead of every chunk
  float* state;      // request r, head h: state + slot_ids[r] * state_stride + state_offset + h * N * P
  size_t state_stride, state_offset;
  const int* span_req;    // [chunks]
  const int* span_start;  // [chunks] first token, counted from the request's first of this step
  const int* span_first;  // [requests] a request's first chunk
  const int* seq_start;
  const int* seq_len;
  const int* slot_ids;
  int n_chunks, n_requests, H, Hk, N, P;
  const float* norm_w;  // head h's P weights at norm_w + h * norm_stride
  int norm_stride;
  float eps;
  const float* gate;  // [rows, ldg], head h at column h * P, or null
  int ldg;
  void* out;
  int ldo, out_dtype;
  int gate_sigmoid;  // the gate passes a sigmoid instead of a silu
  // a decay per key channel (null: one a head)
  float* k_end;   // [rows, H * Np] exp(L_C - L_t) k_t
  float* q_hat;   // [rows, H * Np] exp(L_t) q_t
  float* scores;  // [chunks, H, 64, 64] q_t . k_j with the decays between, 0 above the diagonal
  float* shrink;  // [chunks, H, Np] exp(L_C)
};


// Scores of the rows of tile `wave` against the rows of the tiles up to its own: acc[j] for tile j.
__device__ __forceinline__ void row_products(const float* __restrict__ arow, const float* __restrict__ kb, int ldk, int n,
                                             int Np, int wave, int lr, int lg, f32x4_t acc[4]) {
  const float* brow[4];
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) brow[jt] = kb + (size_t)min(16 * jt + lr, n - 1) * ldk + 4 * lg, acc[jt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int c = 0; c < Np; c += 16) {
    const float4 av = *(const float4*)(arow + c + 4 * lg);
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      if (jt > wave) continue;  // (the same for the whole wave)
      const float4 bv = *(const float4*)(brow[jt] + c);
      acc[jt] = MFMA(av.x, bv.x, acc[jt]);
      acc[jt] = MFMA(av.y, bv.y, acc[jt]);
      acc[jt] = MFMA(av.z, bv.z, acc[jt]);
      acc[jt] = MFMA(av.w, bv.w, acc[jt]);
    }
  }
}

// Tm = (1 + A)^-1 for A strictly lower triangular (Tm zeroed, all of A written, by all threads)
__device__ __forceinline__ void invert_unit_lower(const float* A, float* Tm, float (*tmp)[16 * SS], int wave, int lane, int lr, int lg) {
  __syncthreads();
  // the blocks of sixteen on the diagonal column by column, a lane a column ...
  if (lane < 16) {
    const float* D = A + (16 * wave) * CS + 16 * wave;
    float x[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      float s = t == lane ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < t; ++j) s -= D[t * CS + j] * x[j];
      x[t] = s;
      Tm[(16 * wave + t) * CS + 16 * wave + lane] = s;
    }
  }
  __syncthreads();
  // ... then the blocks d below it: T_ij = -T_ii sum_(j <= m < i) A_im T_mj
  for (int d = 1; d < 4; ++d) {
    const int i = wave, j = wave - d;
    f32x4_t s = {0.f, 0.f, 0.f, 0.f};
    if (j >= 0) {
      for (int m = j; m < i; ++m)
#pragma unroll
        for (int st = 0; st < 4; ++st)
          s = MFMA(A[(16 * i + lr) * CS + 16 * m + 4 * st + lg], Tm[(16 * m + 4 * st + lg) * CS + 16 * j + lr], s);
#pragma unroll
      for (int x = 0; x < 4; ++x) tmp[wave][(4 * lg + x) * SS + lr] = s[x];
    }
    __syncthreads();
    if (j >= 0) {
      s = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int st = 0; st < 4; ++st) s = MFMA(Tm[(16 * i + lr) * CS + 16 * i + 4 * st + lg], tmp[wave][(4 * st + lg) * SS + lr], s);
#pragma unroll
      for (int x = 0; x < 4; ++x) Tm[(16 * i + 4 * lg + x) * CS + 16 * j + lr] = -s[x];
    }
    __syncthreads();
  }
}

__global__ __launch_bounds__(256) void delta_solve_kernel(DeltaChunkArgs a) {
  __shared__ float A[C * CS], Tm[C * CS], tmp[4][16 * SS];
  __shared__ float raw[C], L[C], bt[C], bl[C];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lr = lane & 15, lg = lane >> 4;
  const int h = blockIdx.x, hk = h / (a.H / a.Hk), Np = (a.N + 15) & ~15, Pp = (a.P + 15) & ~15;
  const int r = a.span_req[blockIdx.y], lo = a.span_start[blockIdx.y];
  const int n = min(C, a.seq_len[r] - lo);
  const size_t row0 = (size_t)(a.seq_start[r] + lo);
  const int ldk = a.Hk * Np;
  const float* kb = a.k + row0 * ldk + (size_t)hk * Np;
  if (tid < C) {
    raw[tid] = tid < n ? a.log_g[(row0 + tid) * a.H + h] : 0.f;
    bt[tid] = tid < n ? a.beta[(row0 + tid) * a.H + h] : 0.f;
  }
  for (int e = tid; e < C * CS; e += 256) Tm[e] = 0.f;
  f32x4_t acc[4];
  row_products(kb + (size_t)min(16 * wave + lr, n - 1) * ldk, kb, ldk, n, Np, wave, lr, lg, acc);
  __syncthreads();
  if (tid < C) {
    float s = 0.f;
    for (int t = 0; t <= tid; ++t) s += raw[t];
    L[tid] = s, bl[tid] = bt[tid] * expf(s);
    if (tid < n) a.cum[(row0 + tid) * a.H + h] = s;
  }
  __syncthreads();
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
    if (jt > wave) continue;
    const int j = 16 * jt + lr;
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int t = 16 * wave + 4 * lg + x;
      A[t * CS + j] = j < t && t < n ? bt[t] * expf(L[t] - L[j]) * acc[jt][x] : 0.f;
    }
  }
  invert_unit_lower(A, Tm, tmp, wave, lane, lr, lg);
  // W and U_0, a wave sixteen columns of all 64 rows at a time
  const int nw = Np / 16, nv = Pp / 16;
  for (int ct = wave; ct < nw + nv; ct += 4) {
    const bool is_w = ct < nw;
    const int ld = is_w ? ldk : a.H * Pp;
    const float* src = is_w ? kb + 16 * ct : a.v + row0 * ld + (size_t)h * Pp + 16 * (ct - nw);
    const float* f = is_w ? bl : bt;
    float b[16];
#pragma unroll
    for (int s = 0; s < 16; ++s) b[s] = src[(size_t)min(4 * s + lg, n - 1) * ld + lr];
#pragma unroll
    for (int s = 0; s < 16; ++s) b[s] *= f[4 * s + lg];  // (zero from n on)
    float* dst = is_w ? a.w + row0 * a.H * Np + (size_t)h * Np + 16 * ct : a.u + row0 * a.H * Pp + (size_t)h * Pp + 16 * (ct - nw);
    const size_t ldd = (size_t)a.H * (is_w ? Np : Pp);
#pragma unroll
    for (int tt = 0; tt < 4; ++tt) {
      f32x4_t o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < 4 * (tt + 1); ++s) o = MFMA(Tm[(16 * tt + lr) * CS + 4 * s + lg], b[s], o);
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const int t = 16 * tt + 4 * lg + x;
        if (t < n) dst[t * ldd + lr] = o[x];
      }
    }
  }
}

#define FAR_APART 60.0f  // how far log g may fall within eight tokens for one reference in the middle of sixteen

// (L is kept in units of log 2: the hardware's exponential is that of 2)
#define LOG2E 1.4426950408889634f
__device__ __forceinline__ float exp_2(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float4 exp_diff(const float4& a, const float4& b) {
  return make_float4(exp_2(a.x - b.x), exp_2(a.y - b.y), exp_2(a.z - b.z), exp_2(a.w - b.w));
}
__device__ __forceinline__ float4 mul4(const float4& a, const float4& b) { return make_float4(a.x * b.x, a.y * b.y, a.z * b.z, a.w * b.w); }

__global__ __launch_bounds__(256) void delta_solve_channel_kernel(DeltaChunkArgs a) {
  extern __shared__ __attribute__((aligned(16))) float Ls[];  // [C + 1][Np + 4]: L / log 2, row 0 before the first token
  __shared__ float A[C * CS], Tm[C * CS], tmp[4][16 * SS], bt[C];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lr = lane & 15, lg = lane >> 4;
  const int h = blockIdx.x, hk = h / (a.H / a.Hk), Np = (a.N + 15) & ~15, Pp = (a.P + 15) & ~15, LS = Np + 4;
  const int r = a.span_req[blockIdx.y], lo = a.span_start[blockIdx.y];
  const int n = min(C, a.seq_len[r] - lo);
  const size_t row0 = (size_t)(a.seq_start[r] + lo), ldh = (size_t)a.H * Np;
  const int ldk = a.Hk * Np;
  const float* kb = a.k + row0 * ldk + (size_t)hk * Np;
  const float* qb = a.q + row0 * ldk + (size_t)hk * Np;
  const float* gb = a.log_g + row0 * ldh + (size_t)h * Np;
  if (tid < C) bt[tid] = tid < n ? a.beta[(row0 + tid) * a.H + h] : 0.f;
  for (int e = tid; e < C * CS; e += 256) Tm[e] = 0.f;
  for (int c = tid; c < Np; c += 256) {
    float s = 0.f;
    Ls[c] = 0.f;
    for (int t0 = 0; t0 < C; t0 += 16) {
      float g[16];
#pragma unroll
      for (int i = 0; i < 16; ++i) g[i] = gb[(size_t)min(t0 + i, n - 1) * ldh + c];
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        if (t0 + i < n) s += g[i];
        Ls[(t0 + i + 1) * LS + c] = s * LOG2E;
      }
    }
    a.shrink[((size_t)blockIdx.y * a.H + h) * Np + c] = expf(s);
  }
  __syncthreads();
  // scores of the rows of tile `wave` against the tiles up to its own
  f32x4_t kk[4], qk[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) kk[j] = qk[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  const int t_row = 16 * wave + lr;
  const float* krow = kb + (size_t)min(t_row, n - 1) * ldk + 4 * lg;
  const float* qrow = qb + (size_t)min(t_row, n - 1) * ldk + 4 * lg;
  const float* lrow = Ls + (t_row + 1) * LS + 4 * lg;
  const float* l_ahead = Ls + 16 * wave * LS + 4 * lg;        // L ahead of this tile
  const float* l_mid = Ls + (16 * wave + 8) * LS + 4 * lg;    // in its middle
  const float* l_last = Ls + (16 * wave + 16) * LS + 4 * lg;  // at its end
  float fall = 0.f;
  for (int c = 0; c < Np; c += 16) {
    const float4 kv = *(const float4*)(krow + c), qv = *(const float4*)(qrow + c), lt = *(const float4*)(lrow + c);
    const float4 la = *(const float4*)(l_ahead + c), lm = *(const float4*)(l_mid + c), le = *(const float4*)(l_last + c);
    fall = fmaxf(fall, fmaxf(fmaxf(la.x - lm.x, la.y - lm.y), fmaxf(la.z - lm.z, la.w - lm.w)));
    fall = fmaxf(fall, fmaxf(fmaxf(lm.x - le.x, lm.y - le.y), fmaxf(lm.z - le.z, lm.w - le.w)));
    const float4 down = exp_diff(lt, la), kd = mul4(kv, down), qd = mul4(qv, down);
#pragma unroll
    for (int jt = 0; jt < 3; ++jt) {
      if (jt >= wave) continue;  // (the same for the whole wave)
      const int j = 16 * jt + lr;
      const float4 kj = *(const float4*)(kb + (size_t)min(j, n - 1) * ldk + 4 * lg + c);
      const float4 b = mul4(kj, exp_diff(la, *(const float4*)(Ls + (j + 1) * LS + 4 * lg + c)));
      kk[jt] = MFMA(kd.x, b.x, kk[jt]), kk[jt] = MFMA(kd.y, b.y, kk[jt]);
      kk[jt] = MFMA(kd.z, b.z, kk[jt]), kk[jt] = MFMA(kd.w, b.w, kk[jt]);
      qk[jt] = MFMA(qd.x, b.x, qk[jt]), qk[jt] = MFMA(qd.y, b.y, qk[jt]);
      qk[jt] = MFMA(qd.z, b.z, qk[jt]), qk[jt] = MFMA(qd.w, b.w, qk[jt]);
    }
    // (entries above the diagonal may overflow here; they are not used)
    const float4 dm = exp_diff(lt, lm), km = mul4(kv, dm), qm = mul4(qv, dm), b = mul4(kv, exp_diff(lm, lt));
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      if (jt != wave) continue;
      kk[jt] = MFMA(km.x, b.x, kk[jt]), kk[jt] = MFMA(km.y, b.y, kk[jt]);
      kk[jt] = MFMA(km.z, b.z, kk[jt]), kk[jt] = MFMA(km.w, b.w, kk[jt]);
      qk[jt] = MFMA(qm.x, b.x, qk[jt]), qk[jt] = MFMA(qm.y, b.y, qk[jt]);
      qk[jt] = MFMA(qm.z, b.z, qk[jt]), qk[jt] = MFMA(qm.w, b.w, qk[jt]);
    }
  }
  if (wave_max(fall) > FAR_APART * LOG2E) {  // (the whole wave) pair by pair: four rows of this lane's column
    const float* kj = kb + (size_t)min(t_row, n - 1) * ldk;
    const float* lj = Ls + (t_row + 1) * LS;
    const float* kt[4];
    const float* qt[4];
    const float* ltp[4];
    float sk[4] = {0.f, 0.f, 0.f, 0.f}, sq[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int t = min(16 * wave + 4 * lg + x, n - 1);
      kt[x] = kb + (size_t)t * ldk, qt[x] = qb + (size_t)t * ldk, ltp[x] = Ls + (16 * wave + 4 * lg + x + 1) * LS;
    }
    for (int c = 0; c < a.N; ++c) {
      const float kv = kj[c], lv = lj[c];
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const float e = kv * exp_2(fminf(ltp[x][c] - lv, 0.f));
        sk[x] += kt[x][c] * e, sq[x] += qt[x][c] * e;
      }
    }
#pragma unroll
    for (int jt = 0; jt < 4; ++jt)
      if (jt == wave)
#pragma unroll
        for (int x = 0; x < 4; ++x) kk[jt][x] = sk[x], qk[jt][x] = sq[x];
  }
  float* at = a.scores + ((size_t)blockIdx.y * a.H + h) * C * C;
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
    const int j = 16 * jt + lr;
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int t = 16 * wave + 4 * lg + x;
      A[t * CS + j] = j < t && t < n ? bt[t] * kk[jt][x] : 0.f;
      at[t * C + j] = j <= t && t < n ? qk[jt][x] : 0.f;
    }
  }
  invert_unit_lower(A, Tm, tmp, wave, lane, lr, lg);
  // W, U_0 and the scaled keys and queries, a wave sixteen columns of all 64 rows at a time
  const int nw = Np / 16, nv = Pp / 16;
  for (int ct = wave; ct < nw + nv; ct += 4) {
    const bool is_w = ct < nw;
    const int ld = is_w ? ldk : a.H * Pp;
    const float* src = is_w ? kb + 16 * ct : a.v + row0 * ld + (size_t)h * Pp + 16 * (ct - nw);
    float b[16];
#pragma unroll
    for (int s = 0; s < 16; ++s) b[s] = src[(size_t)min(4 * s + lg, n - 1) * ld + lr];
    if (is_w) {
      const size_t col = (size_t)h * Np + 16 * ct + lr;
      const float* lc = Ls + 16 * ct + lr;
      const float end = lc[C * LS];
      float q[16];
#pragma unroll
      for (int s = 0; s < 16; ++s) q[s] = qb[(size_t)min(4 * s + lg, n - 1) * ldk + 16 * ct + lr];
#pragma unroll
      for (int s = 0; s < 16; ++s) {
        const int t = 4 * s + lg;
        const float l = lc[(t + 1) * LS], down = exp_2(l);
        if (t < n) a.k_end[(row0 + t) * ldh + col] = b[s] * exp_2(end - l), a.q_hat[(row0 + t) * ldh + col] = q[s] * down;
        b[s] *= bt[t] * down;  // (bt is zero from n on)
      }
    } else {
#pragma unroll
      for (int s = 0; s < 16; ++s) b[s] *= bt[4 * s + lg];
    }
    float* dst = is_w ? a.w + row0 * ldh + (size_t)h * Np + 16 * ct : a.u + row0 * a.H * Pp + (size_t)h * Pp + 16 * (ct - nw);
    const size_t ldd = (size_t)a.H * (is_w ? Np : Pp);
#pragma unroll
    for (int tt = 0; tt < 4; ++tt) {
      f32x4_t o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < 4 * (tt + 1); ++s) o = MFMA(Tm[(16 * tt + lr) * CS + 4 * s + lg], b[s], o);
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const int t = 16 * tt + 4 * lg + x;
        if (t < n) dst[t * ldd + lr] = o[x];
      }
    }
  }
}

// NT: tiles of sixteen key columns a wave
// BY: a decay per key channel
template <int NT, bool BY>
__global__ __launch_bounds__(256) void delta_states_kernel(DeltaChunkArgs a) {
  __shared__ float Ss[NT * 64 * SS], Us[C * SS];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lr = lane & 15, lg = lane >> 4;
  const int h = blockIdx.x, r = blockIdx.y, p0 = blockIdx.z * 16, hk = h / (a.H / a.Hk);
  const int N = a.N, P = a.P, Np = (N + 15) & ~15, Pp = (P + 15) & ~15, NC = Np / 16;
  const int len = a.seq_len[r], n_chunks = (len + C - 1) / C, first = a.span_first[r];
  const size_t base = (size_t)a.seq_start[r];
  float* Sg = a.state + (size_t)a.slot_ids[r] * a.state_stride + a.state_offset + (size_t)h * N * P;
  const int p = p0 + lr, ldk = a.Hk * Np;
  const size_t ldw = (size_t)a.H * Np, ldu = (size_t)a.H * Pp;
  f32x4_t S[NT];
#pragma unroll
  for (int q = 0; q < NT; ++q)
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int i = 16 * (wave + 4 * q) + 4 * lg + x;
      const float s = Sg[(size_t)min(i, N - 1) * P + min(p, P - 1)];
      S[q][x] = i < N && p < P ? s : 0.f;
    }
  // a chunk's operands, asked for a chunk ahead
  float4 wf[4 * NT];
  float kf[NT][16], uf[4], lt[4], le = 0.f;
  float4 sh[NT];  // what the rows of S shrink by (BY)
  const int t_row = 16 * wave + lr;  // this lane's row of W
  auto rows_of = [&](int c) { return min(C, len - c * C); };
  auto load_w = [&](int c) {
    const int n = rows_of(c);
    const float* wr = a.w + (base + c * C + min(t_row, n - 1)) * ldw + (size_t)h * Np + 4 * lg;
#pragma unroll
    for (int i = 0; i < 4 * NT; ++i) wf[i] = *(const float4*)(wr + 16 * min(i, NC - 1));
  };
  auto load_u = [&](int c) {
    const int n = rows_of(c);
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const size_t row = base + c * C + min(16 * wave + 4 * lg + x, n - 1);
      uf[x] = a.u[row * ldu + (size_t)h * Pp + p];
      if (!BY) lt[x] = a.cum[row * a.H + h];
    }
    if (!BY) le = a.cum[(base + c * C + n - 1) * a.H + h];
  };
  auto load_k = [&](int c) {
    const int n = rows_of(c);
#pragma unroll
    for (int q = 0; q < NT; ++q)
#pragma unroll
      for (int s = 0; s < 16; ++s)
        kf[q][s] = BY ? a.k_end[(base + c * C + min(4 * s + lg, n - 1)) * ldw + (size_t)h * Np + 16 * min(wave + 4 * q, NC - 1) + lr]
                      : a.k[(base + c * C + min(4 * s + lg, n - 1)) * ldk + (size_t)hk * Np + 16 * min(wave + 4 * q, NC - 1) + lr];
    if constexpr (BY) {
#pragma unroll
      for (int q = 0; q < NT; ++q)
        sh[q] = *(const float4*)(a.shrink + ((size_t)(first + c) * a.H + h) * Np + 16 * min(wave + 4 * q, NC - 1) + 4 * lg);
    }
  };
  load_w(0), load_u(0), load_k(0);
  for (int c = 0; c < n_chunks; ++c) {
    const int n = rows_of(c), next = min(c + 1, n_chunks - 1);
    float* ahead = a.states + ((size_t)(first + c) * a.H + h) * Np * Pp;
    if (c > 0) __syncthreads();  // the chunk before is done with Ss and Us
#pragma unroll
    for (int q = 0; q < NT; ++q)
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const int i = 16 * (wave + 4 * q) + 4 * lg + x;
        if (i < Np) Ss[i * SS + lr] = S[q][x], ahead[(size_t)i * Pp + p] = S[q][x];
      }
    __syncthreads();
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4 * NT; ++i) {
      if (i >= NC) continue;  // (the same for the whole block)
      const float* sr = Ss + (16 * i + 4 * lg) * SS + lr;
      acc = MFMA(wf[i].x, sr[0], acc);
      acc = MFMA(wf[i].y, sr[SS], acc);
      acc = MFMA(wf[i].z, sr[2 * SS], acc);
      acc = MFMA(wf[i].w, sr[3 * SS], acc);
    }
    load_w(next);
    const float l_end = le;
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int t = 16 * wave + 4 * lg + x;
      const float u = uf[x] - acc[x];
      if (t < n) a.u[(base + c * C + t) * ldu + (size_t)h * Pp + p] = u;
      Us[t * SS + lr] = t < n ? (BY ? u : u * expf(l_end - lt[x])) : 0.f;
    }
    if (next != c) load_u(next);
    __syncthreads();
    const float shrink = BY ? 1.f : expf(l_end);
#pragma unroll
    for (int q = 0; q < NT; ++q) {
      if constexpr (BY) S[q] *= f32x4_t{sh[q].x, sh[q].y, sh[q].z, sh[q].w};
      else S[q] *= shrink;
#pragma unroll
      for (int s = 0; s < 16; ++s) S[q] = MFMA(kf[q][s], Us[(4 * s + lg) * SS + lr], S[q]);
    }
    load_k(next);
  }
#pragma unroll
  for (int q = 0; q < NT; ++q)
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int i = 16 * (wave + 4 * q) + 4 * lg + x;
      if (i < N && p < P) Sg[(size_t)i * P + p] = S[q][x];
    }
}

// CT: tiles of sixteen value columns a wave
template <typename T, int CT, bool BY>
__global__ __launch_bounds__(256) void delta_outputs_kernel(DeltaChunkArgs a) {
  extern __shared__ __attribute__((aligned(16))) float Q[];  // [C][Np + 4]
  __shared__ float AT[C * CS], L[C], ss[4][C];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lr = lane & 15, lg = lane >> 4;
  const int h = blockIdx.x, hk = h / (a.H / a.Hk), P = a.P, Np = (a.N + 15) & ~15, Pp = (P + 15) & ~15, QS = Np + 4;
  const int r = a.span_req[blockIdx.y], lo = a.span_start[blockIdx.y];
  const int n = min(C, a.seq_len[r] - lo);
  const size_t row0 = (size_t)(a.seq_start[r] + lo);
  const int ldk = a.Hk * Np;
  const float* kb = a.k + row0 * ldk + (size_t)hk * Np;
  const int ldq = BY ? a.H * Np : ldk;
  const float* qb = BY ? a.q_hat + row0 * ldq + (size_t)h * Np : a.q + row0 * ldk + (size_t)hk * Np;
  for (int e = tid; e < C * Np / 4; e += 256) {
    const int t = e / (Np / 4), c = (e - t * (Np / 4)) * 4;
    *(float4*)(Q + t * QS + c) = *(const float4*)(qb + (size_t)min(t, n - 1) * ldq + c);
  }
  if (BY) {
    const float* at = a.scores + ((size_t)blockIdx.y * a.H + h) * C * C;
    for (int e = tid; e < C * C / 4; e += 256) *(float4*)(AT + (e / (C / 4)) * CS + 4 * (e % (C / 4))) = *(const float4*)(at + 4 * e);
  }
  if (!BY && tid < C) L[tid] = a.cum[(row0 + min(tid, n - 1)) * a.H + h];
  __syncthreads();
  if constexpr (!BY) {
    f32x4_t acc[4];
    row_products(Q + (16 * wave + lr) * QS, kb, ldk, n, Np, wave, lr, lg, acc);
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      if (jt > wave) continue;
      const int j = 16 * jt + lr;
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const int t = 16 * wave + 4 * lg + x;
        AT[t * CS + j] = j <= t && t < n ? expf(L[t] - L[j]) * acc[jt][x] : 0.f;
      }
    }
    __syncthreads();
  }
  const size_t ldu = (size_t)a.H * Pp;
  const float* S0 = a.states + ((size_t)blockIdx.y * a.H + h) * Np * Pp;
  f32x4_t o[CT][4];
#pragma unroll
  for (int ci = 0; ci < CT; ++ci) {
    const int ct = wave + 4 * ci;
#pragma unroll
    for (int tt = 0; tt < 4; ++tt) o[ci][tt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (16 * ct >= Pp) continue;  // (the same for the whole wave)
    const int p = 16 * ct + lr;
    float b[16];
#pragma unroll
    for (int s = 0; s < 16; ++s) {
      const float u = a.u[(row0 + min(4 * s + lg, n - 1)) * ldu + (size_t)h * Pp + p];
      b[s] = 4 * s + lg < n ? u : 0.f;
    }
    // exp(L_t) Q S_0 first, then the chunk's own tokens on top
#pragma unroll 2
    for (int c = 0; c < Np; c += 16) {
      const float* sr = S0 + (size_t)(c + 4 * lg) * Pp + p;
      const float s0 = sr[0], s1 = sr[Pp], s2 = sr[2 * Pp], s3 = sr[3 * Pp];
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) {
        const float4 qv = *(const float4*)(Q + (16 * tt + lr) * QS + c + 4 * lg);
        o[ci][tt] = MFMA(qv.x, s0, o[ci][tt]);
        o[ci][tt] = MFMA(qv.y, s1, o[ci][tt]);
        o[ci][tt] = MFMA(qv.z, s2, o[ci][tt]);
        o[ci][tt] = MFMA(qv.w, s3, o[ci][tt]);
      }
    }
#pragma unroll
    for (int tt = 0; tt < 4; ++tt) {
#pragma unroll
      for (int x = 0; x < 4; ++x)
        if (!BY) o[ci][tt][x] *= expf(L[16 * tt + 4 * lg + x]);
#pragma unroll
      for (int s = 0; s < 4 * (tt + 1); ++s) o[ci][tt] = MFMA(AT[(16 * tt + lr) * CS + 4 * s + lg], b[s], o[ci][tt]);
    }
  }
  // the root mean square over the head (columns beyond P are zero)
#pragma unroll
  for (int tt = 0; tt < 4; ++tt)
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      float q = 0.f;
#pragma unroll
      for (int ci = 0; ci < CT; ++ci) q += o[ci][tt][x] * o[ci][tt][x];
      q = group_sum<16>(q);
      if (lr == 0) ss[wave][16 * tt + 4 * lg + x] = q;
    }
  __syncthreads();
#pragma unroll
  for (int tt = 0; tt < 4; ++tt)
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int t = 16 * tt + 4 * lg + x;
      if (t >= n) continue;
      const float rstd = 1.0f / sqrtf(((ss[0][t] + ss[1][t]) + (ss[2][t] + ss[3][t])) / (float)P + a.eps);
#pragma unroll
      for (int ci = 0; ci < CT; ++ci) {
        const int p = 16 * (wave + 4 * ci) + lr;
        if (p >= P) continue;
        float v = o[ci][tt][x] * rstd * a.norm_w[(size_t)h * a.norm_stride + p];
        if (a.gate) {
          const float z = a.gate[(row0 + t) * a.ldg + (size_t)h * P + p];
          v *= a.gate_sigmoid ? sigmoid_f(z) : silu_f(z);
        }
        ((T*)a.out)[(row0 + t) * a.ldo + (size_t)h * P + p] = from_f32<T>(v);
      }
    }
}

struct LowRankGates {
  const float* u;  // [rows, ldu]
  int ldu, n_rows;
  int a_col, a_rank;  // the decay's middle: columns a_col .. of u (a multiple of 4), a_rank of them (of 8)
  const void* a2;     // [H N][a_rank]
  const float* A_log;    // [H]
  const float* dt_bias;  // [H N]
  float* log_g;          // [rows, H * Np]
  int g_col, g_rank;  // the gate's middle
  const void* g2;     // [H P][g_rank], or null: no gate
  float* gate;        // [rows, H * P]
  int H, N, P, dtype;
};

// Block (64 tokens, 64 columns of log g or of the gate): a wave sixteen tokens of all columns.
template <typename T>
__global__ __launch_bounds__(256) void lowrank_gates_kernel(LowRankGates p, int decay_tiles) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lr = lane & 15, lg = lane >> 4;
  const bool decay = (int)blockIdx.y < decay_tiles;
  const int c0 = 64 * (decay ? blockIdx.y : blockIdx.y - decay_tiles), total = p.H * (decay ? p.N : p.P);
  const int rank = decay ? p.a_rank : p.g_rank, row0 = 64 * blockIdx.x + 16 * wave;
  const T* w2 = (const T*)(decay ? p.a2 : p.g2);
  const float* row = p.u + (size_t)min(row0 + lr, p.n_rows - 1) * p.ldu + (decay ? p.a_col : p.g_col);
  const T* w[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) w[j] = w2 + (size_t)min(c0 + 16 * j + lr, total - 1) * rank;
  f32x4_t acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) acc[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  rows_product<4>([&](int k) { return *(const float4*)(row + k); }, w, rank, 0, 1, acc);
  const int Np = (p.N + 15) & ~15;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int c = c0 + 16 * j + lr;
    if (c >= total) continue;
    const int h = decay ? c / p.N : 0;
    const float rate = decay ? expf(p.A_log[h]) : 0.f, bias = decay ? p.dt_bias[c] : 0.f;
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int t = row0 + 4 * lg + x;
      if (t >= p.n_rows) continue;
      if (decay) p.log_g[(size_t)t * p.H * Np + h * Np + (c - h * p.N)] = -rate * softplus_f(acc[j][x] + bias);
      else p.gate[(size_t)t * total + c] = acc[j][x];
    }
  }
  // the padding between heads: columns that no key has do not decay
  if (decay && Np != p.N && blockIdx.y == 0) {
    const int pad = Np - p.N;
    for (int e = threadIdx.x; e < 64 * p.H * pad; e += 256) {
      const int t = 64 * blockIdx.x + e / (p.H * pad), i = e % (p.H * pad);
      if (t < p.n_rows) p.log_g[(size_t)t * p.H * Np + (i / pad) * Np + p.N + i % pad] = 0.f;
    }
  }
}

DEFINE_LAST_ERROR(mlxlm_last_error)

extern "C" int delta_prepare(const DeltaPrepareArgs* args, hipStream_t stream) {
  const DeltaPrepareArgs& a = *args;
  if (a.n_rows <= 0) return 0;
  if (!a.u || !a.conv_w || (a.log_g && (!a.A_log || !a.dt_bias)) || !a.state || !a.token_req || !a.positions || !a.seq_start || !a.seq_len ||
      !a.slot_ids || !a.q || !a.k || !a.v || !a.beta)
    FAIL("delta_prepare: null pointer");
  if (a.Hk <= 0 || a.H <= 0 || a.H % a.Hk || a.N <= 0 || a.P <= 0 || a.N > PREPARE_MAX || a.P > PREPARE_MAX)
    FAIL("delta_prepare: %d heads over %d key heads, keys of %d and values of %d (at most %d)", a.H, a.Hk, a.N, a.P, PREPARE_MAX);
  const int channels = 2 * a.Hk * a.N + a.H * a.P;
  if (a.taps < 1 || a.b_col < 0 || a.a_col < 0 || a.ldu < channels || a.ldu < a.b_col + a.H || (a.log_g && a.ldu < a.a_col + a.H))
    FAIL("delta_prepare: %d taps over %d channels, gates from columns %d and %d, in rows of %d", a.taps, channels, a.b_col, a.a_col, a.ldu);
  if (a.taps > 1 && a.state_stride < a.ring_offset + (size_t)a.taps * channels) FAIL("delta_prepare: the state rows are too short");
  const int items = 2 * a.Hk + a.H + 1;
  hipLaunchKernelGGL(delta_prepare_kernel, dim3(a.n_rows, (items + 3) / 4), dim3(256), 0, stream, a);
  CHECK_LAUNCH("delta_prepare");
  return 0;
}

// 1 if delta_chunks takes a state of N x P
extern "C" int delta_chunks_takes(int N, int P) { return N > 0 && P > 0 && N <= MAX_N && P <= MAX_P; }

extern "C" int delta_chunks(const DeltaChunkArgs* args, hipStream_t stream) {
  const DeltaChunkArgs& a = *args;
  if (a.n_requests <= 0 || a.n_chunks <= 0 || a.H <= 0) return 0;
  if (!a.q || !a.k || !a.v || !a.log_g || !a.beta || (!a.cum && !a.k_end) || !a.w || !a.u || !a.states || !a.state || !a.span_req ||
      !a.span_start || !a.span_first || !a.seq_start || !a.seq_len || !a.slot_ids || !a.norm_w || !a.out)
    FAIL("delta_chunks: null pointer");
  if (a.Hk <= 0 || a.H % a.Hk) FAIL("delta_chunks: %d heads over %d key heads", a.H, a.Hk);
  if (!delta_chunks_takes(a.N, a.P)) FAIL("delta_chunks: a state of %d x %d (at most %d x %d)", a.N, a.P, MAX_N, MAX_P);
  if (a.ldo < a.H * a.P || (a.gate && a.ldg < a.H * a.P) || (a.norm_stride != 0 && a.norm_stride < a.P))
    FAIL("delta_chunks: a row is narrower than its heads");
  if (a.state_stride < a.state_offset + (size_t)a.H * a.N * a.P) FAIL("delta_chunks: the state rows are too short");
  if (((uintptr_t)a.q | (uintptr_t)a.k | (uintptr_t)a.w) & 15) FAIL("delta_chunks: 16-byte aligned rows");
  if (a.out_dtype != DT_F32 && a.out_dtype != DT_BF16) FAIL("delta_chunks: unknown dtype code %d", a.out_dtype);
  const bool by = a.k_end != nullptr;
  if (by && (!a.q_hat || !a.scores || !a.shrink)) FAIL("delta_chunks: null pointer");
  if (((uintptr_t)a.q_hat | (uintptr_t)a.scores | (uintptr_t)a.shrink) & 15) FAIL("delta_chunks: 16-byte aligned rows");
  const int Np = (a.N + 15) & ~15, Pp = (a.P + 15) & ~15, nt = (Np + 63) / 64, ct = (Pp + 63) / 64;
  const dim3 chunk_grid(a.H, a.n_chunks), state_grid(a.H, a.n_requests, Pp / 16), block(256);
  static bool allowed = false;
  if (by && !allowed) {
    (void)hipFuncSetAttribute((const void*)delta_solve_channel_kernel, hipFuncAttributeMaxDynamicSharedMemorySize,
                              (C + 1) * (MAX_N + 4) * (int)sizeof(float));
    allowed = true;
  }
  if (by) hipLaunchKernelGGL(delta_solve_channel_kernel, chunk_grid, block, (size_t)(C + 1) * (Np + 4) * sizeof(float), stream, a);
  else hipLaunchKernelGGL(delta_solve_kernel, chunk_grid, block, 0, stream, a);
#define STATES(BY)                                                                                             \
  do {                                                                                                         \
    if (nt == 1) hipLaunchKernelGGL((delta_states_kernel<1, BY>), state_grid, block, 0, stream, a);            \
    else if (nt == 2) hipLaunchKernelGGL((delta_states_kernel<2, BY>), state_grid, block, 0, stream, a);       \
    else hipLaunchKernelGGL((delta_states_kernel<4, BY>), state_grid, block, 0, stream, a);                    \
  } while (0)
  if (by) STATES(true);
  else STATES(false);
#undef STATES
  const size_t lds = (size_t)C * (Np + 4) * sizeof(float);
  static bool raised = false;
  if (!raised) {
    const int most = C * (MAX_N + 4) * (int)sizeof(float);
#define RAISE(T, CT)                                                                                                          \
  (void)hipFuncSetAttribute((const void*)delta_outputs_kernel<T, CT, false>, hipFuncAttributeMaxDynamicSharedMemorySize, most); \
  (void)hipFuncSetAttribute((const void*)delta_outputs_kernel<T, CT, true>, hipFuncAttributeMaxDynamicSharedMemorySize, most)
    RAISE(float, 1); RAISE(float, 2); RAISE(float, 4); RAISE(bf16, 1); RAISE(bf16, 2); RAISE(bf16, 4);
#undef RAISE
    raised = true;
  }
#define OUTPUTS(T, BY)                                                                                          \
  do {                                                                                                          \
    if (ct == 1) hipLaunchKernelGGL((delta_outputs_kernel<T, 1, BY>), chunk_grid, block, lds, stream, a);       \
    else if (ct == 2) hipLaunchKernelGGL((delta_outputs_kernel<T, 2, BY>), chunk_grid, block, lds, stream, a);  \
    else hipLaunchKernelGGL((delta_outputs_kernel<T, 4, BY>), chunk_grid, block, lds, stream, a);               \
  } while (0)
  if (a.out_dtype == DT_F32) {
    if (by) OUTPUTS(float, true);
    else OUTPUTS(float, false);
  } else {
    if (by) OUTPUTS(bf16, true);
    else OUTPUTS(bf16, false);
  }
#undef OUTPUTS
  CHECK_LAUNCH("delta_chunks");
  return 0;
}

extern "C" int lowrank_gates(const LowRankGates* args, hipStream_t stream) {
  const LowRankGates& a = *args;
  if (a.n_rows <= 0) return 0;
  if (!a.u || !a.a2 || !a.A_log || !a.dt_bias || !a.log_g || (a.g2 && !a.gate)) FAIL("lowrank_gates: null pointer");
  if (a.H <= 0 || a.N <= 0 || a.P <= 0 || a.ldu % 4 || ((uintptr_t)a.u & 15)) FAIL("lowrank_gates: %d heads of %d and %d, rows of %d", a.H, a.N, a.P, a.ldu);
  if (a.a_rank <= 0 || a.a_rank % 8 || a.a_col < 0 || a.a_col % 4 || a.a_col + a.a_rank > a.ldu)
    FAIL("lowrank_gates: a middle of %d columns at %d in rows of %d", a.a_rank, a.a_col, a.ldu);
  if (a.g2 && (a.g_rank <= 0 || a.g_rank % 8 || a.g_col < 0 || a.g_col % 4 || a.g_col + a.g_rank > a.ldu))
    FAIL("lowrank_gates: a middle of %d columns at %d in rows of %d", a.g_rank, a.g_col, a.ldu);
  if (((uintptr_t)a.a2 | (uintptr_t)a.g2) & 15) FAIL("lowrank_gates: 16-byte aligned matrices");
  const int decay = (a.H * a.N + 63) / 64, gate = a.g2 ? (a.H * a.P + 63) / 64 : 0;
  const dim3 grid((a.n_rows + 63) / 64, decay + gate), block(256);
  if (a.dtype == DT_F32) hipLaunchKernelGGL(lowrank_gates_kernel<float>, grid, block, 0, stream, a, decay);
  else if (a.dtype == DT_BF16) hipLaunchKernelGGL(lowrank_gates_kernel<bf16>, grid, block, 0, stream, a, decay);
  else FAIL("lowrank_gates: unknown dtype code %d", a.dtype);
  CHECK_LAUNCH("lowrank_gates");
  return 0;
}
