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
//                  silu(gate).
//
// All 32-bit, the products on v_mfma_f32_16x16x4_f32 (lane l brings A[l % 16][l / 16] and
// B[l / 16][l % 16] and gets D[4 (l / 16) + x][l % 16]; where both operands run over the same
// columns, a lane brings four consecutive ones to four instructions).
#include "common.h"

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
  float* log_g;  // [rows, H]
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
      a.log_g[(size_t)row0 * a.H + h] = -expf(a.A_log[h]) * softplus_f(ur[a.a_col + h] + a.dt_bias[h]);
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
  const float* log_g;  // [rows, H]
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
  __syncthreads();
  // (1 + A)^-1: the blocks of sixteen on the diagonal column by column, a lane a column ...
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

// NT: tiles of sixteen key columns a wave
template <int NT>
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
  float kf[NT][16], uf[4], lt[4], le;
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
      uf[x] = a.u[row * ldu + (size_t)h * Pp + p], lt[x] = a.cum[row * a.H + h];
    }
    le = a.cum[(base + c * C + n - 1) * a.H + h];
  };
  auto load_k = [&](int c) {
    const int n = rows_of(c);
#pragma unroll
    for (int q = 0; q < NT; ++q)
#pragma unroll
      for (int s = 0; s < 16; ++s)
        kf[q][s] = a.k[(base + c * C + min(4 * s + lg, n - 1)) * ldk + (size_t)hk * Np + 16 * min(wave + 4 * q, NC - 1) + lr];
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
      Us[t * SS + lr] = t < n ? u * expf(l_end - lt[x]) : 0.f;
    }
    if (next != c) load_u(next);
    __syncthreads();
    const float shrink = expf(l_end);
#pragma unroll
    for (int q = 0; q < NT; ++q) {
      S[q] *= shrink;
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
template <typename T, int CT>
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
  const float* qb = a.q + row0 * ldk + (size_t)hk * Np;
  for (int e = tid; e < C * Np / 4; e += 256) {
    const int t = e / (Np / 4), c = (e - t * (Np / 4)) * 4;
    *(float4*)(Q + t * QS + c) = *(const float4*)(qb + (size_t)min(t, n - 1) * ldk + c);
  }
  if (tid < C) L[tid] = a.cum[(row0 + min(tid, n - 1)) * a.H + h];
  __syncthreads();
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
      for (int x = 0; x < 4; ++x) o[ci][tt][x] *= expf(L[16 * tt + 4 * lg + x]);
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
        if (a.gate) v *= silu_f(a.gate[(row0 + t) * a.ldg + (size_t)h * P + p]);
        ((T*)a.out)[(row0 + t) * a.ldo + (size_t)h * P + p] = from_f32<T>(v);
      }
    }
}

DEFINE_LAST_ERROR(mlxlm_last_error)

extern "C" int delta_prepare(const DeltaPrepareArgs* args, hipStream_t stream) {
  const DeltaPrepareArgs& a = *args;
  if (a.n_rows <= 0) return 0;
  if (!a.u || !a.conv_w || !a.A_log || !a.dt_bias || !a.state || !a.token_req || !a.positions || !a.seq_start || !a.seq_len ||
      !a.slot_ids || !a.q || !a.k || !a.v || !a.log_g || !a.beta)
    FAIL("delta_prepare: null pointer");
  if (a.Hk <= 0 || a.H <= 0 || a.H % a.Hk || a.N <= 0 || a.P <= 0 || a.N > PREPARE_MAX || a.P > PREPARE_MAX)
    FAIL("delta_prepare: %d heads over %d key heads, keys of %d and values of %d (at most %d)", a.H, a.Hk, a.N, a.P, PREPARE_MAX);
  const int channels = 2 * a.Hk * a.N + a.H * a.P;
  if (a.taps < 1 || a.b_col < 0 || a.a_col < 0 || a.ldu < channels || a.ldu < a.b_col + a.H || a.ldu < a.a_col + a.H)
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
  if (!a.q || !a.k || !a.v || !a.log_g || !a.beta || !a.cum || !a.w || !a.u || !a.states || !a.state || !a.span_req ||
      !a.span_start || !a.span_first || !a.seq_start || !a.seq_len || !a.slot_ids || !a.norm_w || !a.out)
    FAIL("delta_chunks: null pointer");
  if (a.Hk <= 0 || a.H % a.Hk) FAIL("delta_chunks: %d heads over %d key heads", a.H, a.Hk);
  if (!delta_chunks_takes(a.N, a.P)) FAIL("delta_chunks: a state of %d x %d (at most %d x %d)", a.N, a.P, MAX_N, MAX_P);
  if (a.ldo < a.H * a.P || (a.gate && a.ldg < a.H * a.P) || (a.norm_stride != 0 && a.norm_stride < a.P))
    FAIL("delta_chunks: a row is narrower than its heads");
  if (a.state_stride < a.state_offset + (size_t)a.H * a.N * a.P) FAIL("delta_chunks: the state rows are too short");
  if (((uintptr_t)a.q | (uintptr_t)a.k | (uintptr_t)a.w) & 15) FAIL("delta_chunks: 16-byte aligned rows");
  if (a.out_dtype != DT_F32 && a.out_dtype != DT_BF16) FAIL("delta_chunks: unknown dtype code %d", a.out_dtype);
  const int Np = (a.N + 15) & ~15, Pp = (a.P + 15) & ~15, nt = (Np + 63) / 64, ct = (Pp + 63) / 64;
  const dim3 chunk_grid(a.H, a.n_chunks), state_grid(a.H, a.n_requests, Pp / 16), block(256);
  hipLaunchKernelGGL(delta_solve_kernel, chunk_grid, block, 0, stream, a);
  if (nt == 1) hipLaunchKernelGGL(delta_states_kernel<1>, state_grid, block, 0, stream, a);
  else if (nt == 2) hipLaunchKernelGGL(delta_states_kernel<2>, state_grid, block, 0, stream, a);
  else hipLaunchKernelGGL(delta_states_kernel<4>, state_grid, block, 0, stream, a);
  const size_t lds = (size_t)C * (Np + 4) * sizeof(float);
  static bool raised = false;
  if (!raised) {
    const int most = C * (MAX_N + 4) * (int)sizeof(float);
#define RAISE(T, CT) (void)hipFuncSetAttribute((const void*)delta_outputs_kernel<T, CT>, hipFuncAttributeMaxDynamicSharedMemorySize, most)
    RAISE(float, 1), RAISE(float, 2), RAISE(float, 4), RAISE(bf16, 1), RAISE(bf16, 2), RAISE(bf16, 4);
#undef RAISE
    raised = true;
  }
#define OUTPUTS(T)                                                                                          \
  do {                                                                                                      \
    if (ct == 1) hipLaunchKernelGGL((delta_outputs_kernel<T, 1>), chunk_grid, block, lds, stream, a);       \
    else if (ct == 2) hipLaunchKernelGGL((delta_outputs_kernel<T, 2>), chunk_grid, block, lds, stream, a);  \
    else hipLaunchKernelGGL((delta_outputs_kernel<T, 4>), chunk_grid, block, lds, stream, a);               \
  } while (0)
  if (a.out_dtype == DT_F32) OUTPUTS(float);
  else OUTPUTS(bf16);
#undef OUTPUTS
  CHECK_LAUNCH("delta_chunks");
  return 0;
}
