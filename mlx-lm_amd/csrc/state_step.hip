// A step of few tokens a request through a recurrence over a matrix state, with everything that lies
// between a mixer's projection and its output projection in one launch:
//
//   STEP_DELTA      the gated delta rule on prepared rows (queries scaled, keys of unit length)
//                     u = beta (v - g S^T k);  S <- g S + k u^T;  o = S^T q  (the new S)
//   STEP_DELTA_RAW  the same from the projection's own columns, one token a request: a causal
//                   convolution per channel with silu, queries and keys made unit vectors, beta =
//                   sigmoid(.), g = exp(-exp(A_log) softplus(. + dt_bias)).  The convolution's last
//                   inputs lie in the request's row as a ring, position p in row p % taps: the one
//                   that is written is none of those that are read, so the heads that share a key
//                   head read it side by side.
//   STEP_CHANNEL_RAW  as STEP_DELTA_RAW with a decay per key channel and an output gate through narrow
//                   middles: g[n] = exp(-exp(A_log) softplus(A2 z + dt_bias)), gate = G2 y, with z and y
//                   columns of the projection.
//   STEP_BONUS      a decay per key channel and a bonus for the current token
//                     o = S^T r + (r . (u * k)) v;  S <- diag(w) S + k v^T
//                   with w = exp(-exp(w0 + W2 tanh(z))) made here from the low-rank middle z.
//
// A block a (head, request); S [N][P] lies in the threads' registers, asked for at once and written
// back once (a thread holds every TY-th row of V neighbouring columns), so a step is one trip to
// memory each way.  A token needs one joint reduction over the keys (S^T k and S^T q together: o =
// g S^T q + (q . k) u).  The heads' output is divided by its root mean square (norm weight, a silu or
// sigmoid gate) on the way out.
//
//   lowrank_decay   log w = -exp(w0 + W2 tanh(z)) as rows, for the kernels that take chunks of tokens.
//
// All 32-bit; only `out` may be bfloat16.
#include "common.h"

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

#define UNIT_EPS 1e-6f  // a unit vector is x / sqrt(sum(x^2) + UNIT_EPS)

enum { STEP_DELTA = 0, STEP_DELTA_RAW = 1, STEP_BONUS = 2, STEP_CHANNEL_RAW = 3 };

struct StepArgs {
  const float* q;  // key head hk at column hk * qk_stride, value head h at column h * v_stride
  const float* k;
  const float* v;
  int ldq, ldk, ldv, qk_stride, v_stride;
  const float* gate;  // head h at column h * P, or null
  int ldg;
  const float* norm_w;  // head h's P weights at norm_w + h * norm_stride
  int norm_stride;
  float eps;
  void* out;  // head h at column h * P
  int ldo, out_dtype;
  float* state;  // request r, head h: state + slot_ids[r] * state_stride + state_offset + h * N * P
  size_t state_stride, state_offset;
  const int* seq_start;
  const int* seq_len;
  const int* slot_ids;
  int n_requests, H, Hk, N, P, mode;
  // STEP_DELTA: [tokens, H] each.  STEP_DELTA_RAW: columns of the projection, head h at column h
  const float* log_g;
  const float* beta;
  int ld_gb;
  const float* A_log;
  const float* dt_bias;
  const float* conv_w;  // [2 Hk N + H P channels][taps]: queries, keys, values
  int taps;
  size_t ring_offset;  // [taps][channels] in the request's state row
  const int* positions;
  float q_scale;
  // STEP_BONUS
  const float* z;  // [tokens, rank]
  int ldz, rank, w2_dtype;
  const void* w2t;   // [rank][H N]
  const float* w0;   // [H N]
  const float* bonus;  // [H N]
  int gate_sigmoid;    // the gate passes a sigmoid instead of a silu
  // STEP_CHANNEL_RAW: z and rank as above (rank a multiple of 8), dt_bias [H N]
  const void* a2;  // [H N][rank]
  const float* y;  // [tokens, g_rank] (gate is not read then), or null: no gate, or `gate`
  int ldy, g_rank;
  const void* g2;  // [H P][g_rank]
};

struct Sums3 {
  float a, b, c;
};
__device__ __forceinline__ Sums3 block_sums(Sums3 s, float* red) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
  s.a = wave_sum(s.a), s.b = wave_sum(s.b), s.c = wave_sum(s.c);
  __syncthreads();
  if (lane == 0) red[wave] = s.a, red[16 + wave] = s.b, red[32 + wave] = s.c;
  __syncthreads();
  Sums3 t = {0.f, 0.f, 0.f};
  for (int i = 0; i < nw; ++i) t.a += red[i], t.b += red[16 + i], t.c += red[32 + i];
  return t;
}

template <int V>
struct Cols;
template <>
struct Cols<4> {
  f32x4_t v;
  static __device__ __forceinline__ Cols load(const float* p) { return Cols{*(const f32x4_t*)p}; }
  __device__ __forceinline__ void store(float* p) const { *(f32x4_t*)p = v; }
};
template <>
struct Cols<1> {
  float v;
  static __device__ __forceinline__ Cols load(const float* p) { return Cols{*p}; }
  __device__ __forceinline__ void store(float* p) const { *p = v; }
};

// W2's entry of the low-rank middle
__device__ __forceinline__ float lowrank_logit(const void* w2t, int dtype, const float* tz, int rank, int width, int c) {
  float z = 0.f;
  if (dtype == DT_BF16) {
    const bf16* w = (const bf16*)w2t + c;
#pragma unroll 8
    for (int r = 0; r < rank; ++r) z += to_f32(w[(size_t)r * width]) * tz[r];
  } else {
    const float* w = (const float*)w2t + c;
#pragma unroll 8
    for (int r = 0; r < rank; ++r) z += w[(size_t)r * width] * tz[r];
  }
  return z;
}

// One row of a narrow matrix with a middle in LDS, by sixteen neighbouring lanes; in all of them.
__device__ __forceinline__ float lowrank_row(const bf16* __restrict__ w, const float* m, int rank, int l16) {
  float s = 0.f;
  for (int k = 8 * l16; k < rank; k += 128) {
    const u32x4_t v = *(const u32x4_t*)(w + k);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      s += __uint_as_float(v[i] << 16) * m[k + 2 * i];
      s += __uint_as_float(v[i] & 0xffff0000u) * m[k + 2 * i + 1];
    }
  }
  return group_sum<16>(s);
}
__device__ __forceinline__ float lowrank_row(const float* __restrict__ w, const float* m, int rank, int l16) {
  float s = 0.f;
  for (int k = 4 * l16; k < rank; k += 64) {
    const f32x4_t v = *(const f32x4_t*)(w + k);
#pragma unroll
    for (int i = 0; i < 4; ++i) s += v[i] * m[k + i];
  }
  return group_sum<16>(s);
}
// Up to AHEAD rows a lane group of the two narrow matrices (bfloat16, middles of up to 128 columns), asked
// for before the middles are known.
#define AHEAD 8
__device__ __forceinline__ bool fits_ahead(const StepArgs& a, int threads) {
  return a.w2_dtype == DT_BF16 && a.rank <= 128 && (!a.y || a.g_rank <= 128) && a.N + (a.y ? a.P : 0) <= AHEAD * (threads / 16);
}
template <int TH>
__device__ __forceinline__ void ask_rows(const StepArgs& a, int h, u32x4_t (&w)[AHEAD]) {
  const int k = 8 * (threadIdx.x & 15), total = a.N + (a.y ? a.P : 0);
  const bf16* a2 = (const bf16*)a.a2 + (size_t)h * a.N * a.rank;
  const bf16* g2 = (const bf16*)a.g2 + (size_t)h * a.P * a.g_rank;
#pragma unroll
  for (int i = 0; i < AHEAD; ++i) {
    const int c = threadIdx.x / 16 + i * (TH / 16);
    w[i] = u32x4_t{0u, 0u, 0u, 0u};
    if (c < a.N) {
      if (k < a.rank) w[i] = *(const u32x4_t*)(a2 + (size_t)c * a.rank + k);
    } else if (c < total && k < a.g_rank) {
      w[i] = *(const u32x4_t*)(g2 + (size_t)(c - a.N) * a.g_rank + k);
    }
  }
}
template <int TH>
__device__ __forceinline__ void rows_asked(const StepArgs& a, const u32x4_t (&w)[AHEAD], const float* tz, const float* my, float* ds, float* gs) {
  const int l16 = threadIdx.x & 15, k = 8 * l16, total = a.N + (a.y ? a.P : 0);
  float z[8], y[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) z[j] = k < a.rank ? tz[k + j] : 0.f, y[j] = a.y && k < a.g_rank ? my[k + j] : 0.f;
#pragma unroll
  for (int i = 0; i < AHEAD; ++i) {
    const int c = threadIdx.x / 16 + i * (TH / 16);
    if (c >= total) continue;  // (the same for sixteen lanes)
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      s += __uint_as_float(w[i][j] << 16) * (c < a.N ? z[2 * j] : y[2 * j]);
      s += __uint_as_float(w[i][j] & 0xffff0000u) * (c < a.N ? z[2 * j + 1] : y[2 * j + 1]);
    }
    s = group_sum<16>(s);
    if (l16 == 0) (c < a.N ? ds[c] : gs[c - a.N]) = s;
  }
}
// The decays' logits into ds and the gate's into gs, for head h.
template <typename T, int TH>
__device__ __forceinline__ void lowrank_rows(const StepArgs& a, int h, const float* tz, const float* ty, float* ds, float* gs) {
  const int l16 = threadIdx.x & 15, total = a.N + (a.y ? a.P : 0);
  const T* a2 = (const T*)a.a2 + (size_t)h * a.N * a.rank;
  const T* g2 = (const T*)a.g2 + (size_t)h * a.P * a.g_rank;
#pragma unroll 1
  for (int c = threadIdx.x / 16; c < total; c += TH / 16) {
    if (c < a.N) {
      const float s = lowrank_row(a2 + (size_t)c * a.rank, tz, a.rank, l16);
      if (l16 == 0) ds[c] = s;
    } else {
      const float s = lowrank_row(g2 + (size_t)(c - a.N) * a.g_rank, ty, a.g_rank, l16);
      if (l16 == 0) gs[c - a.N] = s;
    }
  }
}

// V columns a thread, R rows of the state a thread, TH threads
template <int MODE, int V, int R, int TH, typename T>
__global__ __launch_bounds__(TH) void state_step_kernel(StepArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float red[48];
  const int N = a.N, P = a.P, tid = threadIdx.x, h = blockIdx.x, rq = blockIdx.y, group = a.H / a.Hk, hk = h / group;
  const int cols = P / V, TY = min(TH / cols, N), tx = tid % cols, ty = tid / cols;
  const bool active = ty < TY;
  float* part_q = lds;                          // [TY][P]
  float* part_k = part_q + (size_t)TY * P;      // [TY][P] (the delta rule)
  float* us = part_k + (size_t)(MODE == STEP_BONUS ? 0 : TY * P);  // [P]
  float* vs = us + P;                           // [P]
  float* qs = vs + P;                           // [N]
  float* ks = qs + N;                           // [N]
  float* ds = ks + N;                           // [N] the decays (STEP_BONUS)
  float* tz = ds + N;                           // [rank]
  float* gs = tz + a.rank;                      // [P] the gate's logits (STEP_CHANNEL_RAW)
  float* my = gs + P;                           // [g_rank]
  // (raw columns: every request brings one token)
  const int start = a.seq_start[rq], n = MODE == STEP_DELTA_RAW || MODE == STEP_CHANNEL_RAW ? 1 : a.seq_len[rq];
  float* row_state = a.state + (size_t)a.slot_ids[rq] * a.state_stride;
  float* Sg = row_state + a.state_offset + (size_t)h * N * P;
  Cols<V> S[R];
#pragma unroll
  for (int r = 0; r < R; ++r) S[r] = Cols<V>::load(Sg + (size_t)min(ty + TY * r, N - 1) * P + tx * V);

  u32x4_t narrow[AHEAD];
  bool ahead = false;
  if constexpr (MODE == STEP_CHANNEL_RAW && TH <= 512) {
    ahead = fits_ahead(a, TH);
    if (ahead) ask_rows<TH>(a, h, narrow);
  }

  for (int t = 0; t < n; ++t) {
    const size_t row = (size_t)(start + t);
    float gv = a.gate && tid < P ? a.gate[row * a.ldg + (size_t)h * P + tid] : 0.f;
    const float nw = tid < P ? a.norm_w[(size_t)h * a.norm_stride + tid] : 0.f;
    float g = 1.f, beta = 0.f;
    if (t > 0) __syncthreads();  // the token before is done with the arrays
    if constexpr (MODE == STEP_DELTA_RAW || MODE == STEP_CHANNEL_RAW) {
      if constexpr (MODE == STEP_CHANNEL_RAW) {
        for (int i = tid; i < a.rank; i += TH) tz[i] = a.z[row * a.ldz + i];
        if (a.y)
          for (int i = tid; i < a.g_rank; i += TH) my[i] = a.y[row * a.ldy + i];
      }
      const int C = 2 * a.Hk * N + a.H * P, pos = a.positions[row];
      float* ring = row_state + a.ring_offset;
      const bool keeps_keys = h % group == 0;
      for (int c = tid; c < 2 * N + P; c += TH) {
        const int kind = c < N ? 0 : c < 2 * N ? 1 : 2, i = c - kind * N;
        const int ch = kind == 0 ? hk * N + i : kind == 1 ? a.Hk * N + hk * N + i : 2 * a.Hk * N + h * P + i;
        const float in = kind == 0 ? a.q[row * a.ldq + (size_t)hk * N + i]
                                   : kind == 1 ? a.k[row * a.ldk + (size_t)hk * N + i] : a.v[row * a.ldv + (size_t)h * P + i];
        const float* w = a.conv_w + (size_t)ch * a.taps;
        float acc = 0.f;
        for (int j = a.taps - 1; j > 0; --j) {  // the oldest input first
          const float old = ring[(size_t)((pos + a.taps - j) % a.taps) * C + ch];
          acc += w[a.taps - 1 - j] * (pos - j >= 0 ? old : 0.f);
        }
        acc += w[a.taps - 1] * in;
        if (a.taps > 1 && (kind == 2 || keeps_keys)) ring[(size_t)(pos % a.taps) * C + ch] = in;
        (kind == 0 ? qs : kind == 1 ? ks : vs)[i] = silu_f(acc);
      }
      beta = sigmoid_f(a.beta[row * a.ld_gb + h]);
      if constexpr (MODE == STEP_DELTA_RAW) {
        g = expf(-expf(a.A_log[h]) * softplus_f(a.log_g[row * a.ld_gb + h] + a.dt_bias[h]));
      } else {
        __syncthreads();
        if (TH <= 512 && ahead) rows_asked<TH>(a, narrow, tz, my, ds, gs);
        else if (a.w2_dtype == DT_BF16) lowrank_rows<bf16, TH>(a, h, tz, my, ds, gs);
        else lowrank_rows<float, TH>(a, h, tz, my, ds, gs);
        __syncthreads();
        const float rate = expf(a.A_log[h]);
        for (int i = tid; i < N; i += TH) ds[i] = expf(-rate * softplus_f(ds[i] + a.dt_bias[(size_t)h * N + i]));
        if (a.y && tid < P) gv = gs[tid];
      }
    } else {
      for (int i = tid; i < N; i += TH) {
        qs[i] = a.q[row * a.ldq + (size_t)hk * a.qk_stride + i];
        ks[i] = a.k[row * a.ldk + (size_t)hk * a.qk_stride + i];
      }
      for (int c = tid; c < P; c += TH) vs[c] = a.v[row * a.ldv + (size_t)h * a.v_stride + c];
      if constexpr (MODE == STEP_DELTA) {
        beta = a.beta[row * a.ld_gb + h];
        g = expf(a.log_g[row * a.ld_gb + h]);
      } else {
        for (int i = tid; i < a.rank; i += TH) tz[i] = tanhf(a.z[row * a.ldz + i]);
        __syncthreads();
        for (int i = tid; i < N; i += TH) {
          const int c = h * N + i;
          ds[i] = expf(-expf(a.w0[c] + lowrank_logit(a.w2t, a.w2_dtype, tz, a.rank, a.H * N, c)));
        }
      }
    }
    __syncthreads();
    Sums3 s = {0.f, 0.f, 0.f};
    for (int i = tid; i < N; i += TH) {
      const float q = qs[i], k = ks[i];
      if constexpr (MODE == STEP_DELTA_RAW || MODE == STEP_CHANNEL_RAW) s.a += q * q, s.b += k * k;
      s.c += MODE == STEP_BONUS ? q * k * a.bonus[(size_t)h * N + i] : q * k;
    }
    float qf = 1.f, kf = 1.f;  // what queries and keys are still to be multiplied by
    if (active) {
      Cols<V> pq = {}, pk = {};
      Cols<V> vc;
      if constexpr (MODE == STEP_BONUS) vc = Cols<V>::load(vs + tx * V);
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const int i = ty + TY * r;
        if (i < N) {
          if constexpr (MODE == STEP_BONUS) {
            pq.v += qs[i] * S[r].v;
            S[r].v = ds[i] * S[r].v + ks[i] * vc.v;
          } else {
            S[r].v *= MODE == STEP_CHANNEL_RAW ? ds[i] : g;
            pq.v += qs[i] * S[r].v;
            pk.v += ks[i] * S[r].v;
          }
        }
      }
      pq.store(part_q + (size_t)ty * P + tx * V);
      if constexpr (MODE != STEP_BONUS) pk.store(part_k + (size_t)ty * P + tx * V);
    }
    s = block_sums(s, red);  // (its barriers also stand between the partial sums and their readers)
    float dot = s.c;
    if constexpr (MODE == STEP_DELTA_RAW || MODE == STEP_CHANNEL_RAW) {
      qf = a.q_scale / sqrtf(s.a + UNIT_EPS), kf = 1.0f / sqrtf(s.b + UNIT_EPS);
      dot *= qf * kf;
    }
    float o = 0.f;
    if (tid < P) {
      float sq = 0.f, sk = 0.f;
      for (int j = 0; j < TY; ++j) {
        sq += part_q[(size_t)j * P + tid];
        if constexpr (MODE != STEP_BONUS) sk += part_k[(size_t)j * P + tid];
      }
      if constexpr (MODE == STEP_BONUS) {
        o = sq + dot * vs[tid];
      } else {
        const float u = beta * (vs[tid] - kf * sk);
        o = qf * sq + dot * u;
        us[tid] = kf * u;
      }
    }
    if constexpr (MODE != STEP_BONUS) {
      __syncthreads();
      if (active) {
        const Cols<V> uc = Cols<V>::load(us + tx * V);
#pragma unroll
        for (int r = 0; r < R; ++r) {
          const int i = ty + TY * r;
          if (i < N) S[r].v += ks[i] * uc.v;
        }
      }
    }
    const float ss = block_sum(tid < P ? o * o : 0.f, red);
    if (tid < P) {
      o *= nw / sqrtf(ss / (float)P + a.eps);
      if (a.gate || (MODE == STEP_CHANNEL_RAW && a.y)) o *= a.gate_sigmoid ? sigmoid_f(gv) : silu_f(gv);
      ((T*)a.out)[row * a.ldo + (size_t)h * P + tid] = from_f32<T>(o);
    }
  }
  if (active) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int i = ty + TY * r;
      if (i < N) S[r].store(Sg + (size_t)i * P + tx * V);
    }
  }
}

#define DECAY_ROWS 8  // tokens a block

// Block (8 tokens, 256 channels), a thread a channel of all eight.
template <typename T>
__global__ __launch_bounds__(256) void lowrank_decay_kernel(const float* __restrict__ z, int ldz, int rank,
                                                            const T* __restrict__ w2t, const float* __restrict__ w0,
                                                            int width, float* __restrict__ log_w, int n_rows) {
  extern __shared__ float tz[];  // [DECAY_ROWS][rank]
  const int r0 = blockIdx.x * DECAY_ROWS, m = min(DECAY_ROWS, n_rows - r0);
  for (int e = threadIdx.x; e < m * rank; e += 256) tz[e] = tanhf(z[(size_t)(r0 + e / rank) * ldz + e % rank]);
  __syncthreads();
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= width) return;
  float acc[DECAY_ROWS];
  const float base = w0[c];
#pragma unroll
  for (int i = 0; i < DECAY_ROWS; ++i) acc[i] = base;
#pragma unroll 4
  for (int r = 0; r < rank; ++r) {
    const float w = to_f32(w2t[(size_t)r * width + c]);
#pragma unroll
    for (int i = 0; i < DECAY_ROWS; ++i) acc[i] += w * (i < m ? tz[i * rank + r] : 0.f);
  }
#pragma unroll
  for (int i = 0; i < DECAY_ROWS; ++i)
    if (i < m) log_w[(size_t)(r0 + i) * width + c] = -expf(acc[i]);
}

DEFINE_LAST_ERROR(mlxlm_last_error)

#define STEP_MAX_P 256

// The launch for a state of N x P: columns and rows a thread, threads a block; 0 if none fits.
struct StepShape {
  int V, R, TH;
};
static StepShape step_shape(int N, int P) {
  if (N <= 0 || P <= 0 || P > STEP_MAX_P) return StepShape{0, 0, 0};
  const auto rows = [&](int V, int TH) {
    const int ty = TH / (P / V) < N ? TH / (P / V) : N;
    return (N + ty - 1) / ty;
  };
  if (P % 4 == 0) {
    if (rows(4, 256) <= 4) return StepShape{4, 4, 256};
    if (rows(4, 512) <= 8) return StepShape{4, 8, 512};
    if (rows(4, 1024) <= 16) return StepShape{4, 16, 1024};
    if (rows(4, 1024) <= 24) return StepShape{4, 24, 1024};
    return StepShape{0, 0, 0};
  }
  if (rows(1, 256) <= 8) return StepShape{1, 8, 256};
  if (rows(1, 1024) <= 64) return StepShape{1, 64, 1024};
  return StepShape{0, 0, 0};
}

extern "C" int state_step_takes(int N, int P) { return step_shape(N, P).TH > 0; }

template <int MODE, typename T>
static void launch_step(const StepArgs& a, const StepShape& s, size_t lds, hipStream_t stream) {
  const dim3 grid(a.H, a.n_requests);
#define RUN(V, R, TH) hipLaunchKernelGGL((state_step_kernel<MODE, V, R, TH, T>), grid, dim3(TH), lds, stream, a)
  if (s.V == 4 && s.R == 4) RUN(4, 4, 256);
  else if (s.V == 4 && s.R == 8) RUN(4, 8, 512);
  else if (s.V == 4 && s.R == 16) RUN(4, 16, 1024);
  else if (s.V == 4) RUN(4, 24, 1024);
  else if (s.R == 8) RUN(1, 8, 256);
  else RUN(1, 64, 1024);
#undef RUN
}

extern "C" int state_step(const StepArgs* args, hipStream_t stream) {
  const StepArgs& a = *args;
  if (a.n_requests <= 0 || a.H <= 0) return 0;
  if (!a.q || !a.k || !a.v || !a.norm_w || !a.out || !a.state || !a.seq_start || !a.seq_len || !a.slot_ids)
    FAIL("state_step: null pointer");
  if (a.Hk <= 0 || a.H % a.Hk) FAIL("state_step: %d heads over %d key heads", a.H, a.Hk);
  const StepShape s = step_shape(a.N, a.P);
  if (!s.TH) FAIL("state_step: a state of %d x %d is more than a block holds in registers", a.N, a.P);
  if (a.qk_stride < a.N || a.v_stride < a.P || a.ldq < (a.Hk - 1) * a.qk_stride + a.N || a.ldk < (a.Hk - 1) * a.qk_stride + a.N ||
      a.ldv < (a.H - 1) * a.v_stride + a.P || a.ldo < a.H * a.P || (a.gate && a.ldg < a.H * a.P))
    FAIL("state_step: a row is narrower than its heads");
  if (a.norm_stride != 0 && a.norm_stride < a.P) FAIL("state_step: norm weights %d apart for heads of %d", a.norm_stride, a.P);
  if (a.state_stride < a.state_offset + (size_t)a.H * a.N * a.P) FAIL("state_step: the state rows are too short");
  if (s.V == 4 && (a.state_stride % 4 || a.state_offset % 4 || ((uintptr_t)a.state & 15))) FAIL("state_step: the states must be 16-byte aligned");
  if (a.out_dtype != DT_F32 && a.out_dtype != DT_BF16) FAIL("state_step: unknown dtype code %d", a.out_dtype);
  int rank = 0;
  if (a.mode == STEP_DELTA || a.mode == STEP_DELTA_RAW || a.mode == STEP_CHANNEL_RAW) {
    if ((!a.log_g && a.mode != STEP_CHANNEL_RAW) || !a.beta || a.ld_gb < a.H) FAIL("state_step: a decay and a step size for every head");
    if (a.mode == STEP_CHANNEL_RAW) {
      if (!a.z || !a.a2 || a.rank <= 0 || a.rank % 8 || a.ldz < a.rank || a.rank > 2048) FAIL("state_step: decays per key channel from a middle of %d columns (a multiple of 8, at most 2048)", a.rank);
      if (a.y && (!a.g2 || a.g_rank <= 0 || a.g_rank % 8 || a.ldy < a.g_rank || a.g_rank > 2048)) FAIL("state_step: a gate from a middle of %d columns (a multiple of 8, at most 2048)", a.g_rank);
      if (((uintptr_t)a.a2 | (a.y ? (uintptr_t)a.g2 : 0)) & 15) FAIL("state_step: 16-byte aligned matrices");
      if (a.w2_dtype != DT_F32 && a.w2_dtype != DT_BF16) FAIL("state_step: unknown dtype code %d", a.w2_dtype);
      rank = a.rank + a.P + (a.y ? a.g_rank : 0);
    }
    if (a.mode != STEP_DELTA) {
      if (!a.A_log || !a.dt_bias || !a.conv_w || !a.positions || a.taps < 1) FAIL("state_step: null pointer, or %d taps", a.taps);
      if (a.qk_stride != a.N || a.v_stride != a.P) FAIL("state_step: the projection's heads lie side by side");
      if (a.taps > 1 && a.state_stride < a.ring_offset + (size_t)a.taps * (2 * a.Hk * a.N + a.H * a.P))
        FAIL("state_step: the state rows do not hold %d inputs of the convolution", a.taps);
    }
  } else if (a.mode == STEP_BONUS) {
    if (!a.z || !a.w2t || !a.w0 || !a.bonus || a.rank <= 0 || a.ldz < a.rank || a.Hk != a.H)
      FAIL("state_step: decays per key channel from a middle of %d columns", a.rank);
    if (a.w2_dtype != DT_F32 && a.w2_dtype != DT_BF16) FAIL("state_step: unknown dtype code %d", a.w2_dtype);
    if (a.rank > 2048) FAIL("state_step: a middle of %d columns (at most 2048)", a.rank);
    rank = a.rank;
  } else {
    FAIL("state_step: unknown mode %d", a.mode);
  }
  const int cols = a.P / s.V, ty = s.TH / cols < a.N ? s.TH / cols : a.N;
  const size_t lds = ((a.mode == STEP_BONUS ? 1 : 2) * (size_t)ty * a.P + 2 * (size_t)a.P + 3 * (size_t)a.N + rank) * sizeof(float);
  if (lds > 60 * 1024) FAIL("state_step: a state of %d x %d needs %zu bytes of LDS", a.N, a.P, lds);
  const bool f32 = a.out_dtype == DT_F32;
  if (a.mode == STEP_DELTA) {
    if (f32) launch_step<STEP_DELTA, float>(a, s, lds, stream);
    else launch_step<STEP_DELTA, bf16>(a, s, lds, stream);
  } else if (a.mode == STEP_CHANNEL_RAW) {
    if (f32) launch_step<STEP_CHANNEL_RAW, float>(a, s, lds, stream);
    else launch_step<STEP_CHANNEL_RAW, bf16>(a, s, lds, stream);
  } else if (a.mode == STEP_DELTA_RAW) {
    if (f32) launch_step<STEP_DELTA_RAW, float>(a, s, lds, stream);
    else launch_step<STEP_DELTA_RAW, bf16>(a, s, lds, stream);
  } else {
    if (f32) launch_step<STEP_BONUS, float>(a, s, lds, stream);
    else launch_step<STEP_BONUS, bf16>(a, s, lds, stream);
  }
  CHECK_LAUNCH("state_step");
  return 0;
}

// log_w [n_rows, width] = -exp(w0 + tanh(z) W2^T); w2t: W2 transposed, [rank][width], float or bfloat16.
extern "C" int lowrank_decay(const float* z, int ldz, int rank, const void* w2t, int w2_dtype, const float* w0, int width,
                             float* log_w, int n_rows, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  if (!z || !w2t || !w0 || !log_w) FAIL("lowrank_decay: null pointer");
  if (rank <= 0 || rank > 1024 || ldz < rank || width <= 0) FAIL("lowrank_decay: a middle of %d columns (at most 1024) in rows of %d", rank, ldz);
  const dim3 grid((n_rows + DECAY_ROWS - 1) / DECAY_ROWS, (width + 255) / 256), block(256);
  const size_t lds = (size_t)DECAY_ROWS * rank * sizeof(float);
  if (w2_dtype == DT_F32)
    hipLaunchKernelGGL(lowrank_decay_kernel<float>, grid, block, lds, stream, z, ldz, rank, (const float*)w2t, w0, width, log_w, n_rows);
  else if (w2_dtype == DT_BF16)
    hipLaunchKernelGGL(lowrank_decay_kernel<bf16>, grid, block, lds, stream, z, ldz, rank, (const bf16*)w2t, w0, width, log_w, n_rows);
  else
    FAIL("lowrank_decay: unknown dtype code %d", w2_dtype);
  CHECK_LAUNCH("lowrank_decay");
  return 0;
}
