// A feed-forward of many small gated experts of which every token uses a few:
//   router_choice   s = softmax(z) over all router outputs, or the logistic function of each; the `top`
//                   largest of s + correction are chosen (the lower index on a tie), out of all or out
//                   of the best groups of neighbours; their weights are s itself.
//   silu_mul        act = silu(gate) * up for rows [gate | up]   (a dense gated feed-forward)
//   route_and_gate  both of these in one launch, for a step of few tokens whose router, gate and up
//                   came out of one product as float rows
//   expert_rows_up / expert_rows_down
//                   a token's chosen experts read straight from the stacked expert weights, a
//                   wave four features at once: act[t, j, :] = w_tj silu(Wg_e x_t) * (Wu_e x_t) (or
//                   another activation of the two, expert_act), then
//                   y[t, :] += sum_j Wd_e act[t, j, :] + sum_(j: e is an identity expert) w_tj x_t.
//                   Only the chosen experts' weights are read: the kernels for few tokens.  The first
//                   may make the choice itself from the router's outputs, the second (as expert_combine)
//                   may leave the next layer's norm of the rows it completes.
//   expert_tiles    the same for many tokens: the picks are sorted by expert on the device
//                   (expert_sort: counts, offsets, tiles of picks of one expert), and
//                   every tile is a small matrix product on the matrix cores with the rows
//                   gathered through the sorted list (bfloat16: through LDS, tiles of 32, 64 or 128
//                   picks; 32-bit: operands straight from memory): [gate | up] with the activation and
//                   the pick's weight in the epilogue, then down into a row of its own for every
//                   pick; expert_combine adds a token's picks in their order, and the identity
//                   experts' share.  The grid is as large as the tiles could be at most; blocks
//                   beyond the tiles that there are leave at once, so nothing comes to the host.
// The router's softmax, the choice and the weights are 32-bit; products accumulate in 32-bit.
#include "common.h"

__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }

// An expert's activation of its gate and up columns:
//   EXPERT_SILU     silu(g) u
//   EXPERT_CLAMPED  g' sigmoid(1.702 g') (u' + 1)  with g' = min(g, limit), u' = u clamped to [-limit, limit]
enum { EXPERT_SILU = 0, EXPERT_CLAMPED = 1 };
struct ExpertAct {
  int kind;
  float limit;
};
__device__ __forceinline__ float expert_act(const ExpertAct& a, float g, float u) {
  if (a.kind == EXPERT_SILU) return silu_f(g) * u;
  g = fminf(g, a.limit), u = fminf(fmaxf(u, -a.limit), a.limit);
  return g / (1.0f + expf(-1.702f * g)) * (u + 1.0f);
}

// How a token's experts are chosen from its router outputs.
struct RouteArgs {
  const float* z;  // [tokens, ldz], or null: idx and weight hold the choice already
  int ldz;
  const float* correction;  // added to a score for the choice only, or null
  int n_out, renorm;        // renorm: the picks' weights are divided by their sum (+ 1e-20)
  float mult;               // and multiplied by this
  int sigmoid;              // a score is the logistic function of its output instead of the softmax over all
  int groups, keep;         // groups > 1: only outputs of the `keep` best of so many equal groups of neighbours
                            // can be chosen; a group counts the sum of its two largest choice scores
};

// A wave a token, up to ROUTER_PER_LANE outputs a lane.  The k-th pick is the largest choice score
// not picked yet, the lowest index on a tie.
#define ROUTER_PER_LANE 8

// The largest of c over the wave and the lowest index that holds it.
template <int PL>
__device__ __forceinline__ int wave_argmax(const float (&c)[PL], int lane, float* value) {
  float best = -INFINITY;
#pragma unroll
  for (int i = 0; i < PL; ++i) best = fmaxf(best, c[i]);
  best = wave_max(best);
  float first = -1e9f;  // minus the lowest index that holds the best score (indices are exact in a float)
#pragma unroll
  for (int i = PL - 1; i >= 0; --i)
    if (c[i] == best) first = -(float)(lane + 64 * i);
  *value = best;
  return (int)(-wave_max(first));
}

// Choice scores outside the best groups become minus infinity.
template <int PL>
__device__ __forceinline__ void limit_groups(float (&c)[PL], int n_out, int groups, int keep, int lane) {
  const int size = n_out / groups;
  int group[PL];  // of output lane + 64 i
#pragma unroll
  for (int i = 0; i < PL; ++i) group[i] = lane + 64 * i < n_out ? (lane + 64 * i) / size : -1;
  float score[PL];  // group lane + 64 i
#pragma unroll
  for (int i = 0; i < PL; ++i) score[i] = -INFINITY;
  for (int g = 0; g < groups; ++g) {
    float m1 = -INFINITY;
#pragma unroll
    for (int i = 0; i < PL; ++i) {
      if (group[i] == g) m1 = fmaxf(m1, c[i]);
    }
    m1 = wave_max(m1);
    float m2 = -INFINITY;
    int equal = 0;
#pragma unroll
    for (int i = 0; i < PL; ++i) {
      const bool in = group[i] == g;
      equal += __popcll(__ballot(in && c[i] == m1));
      if (in && c[i] != m1) m2 = fmaxf(m2, c[i]);
    }
    m2 = equal > 1 ? m1 : wave_max(m2);
    const float total = size > 1 ? m1 + m2 : m1;
#pragma unroll
    for (int i = 0; i < PL; ++i)
      if (lane + 64 * i == g) score[i] = total;
  }
  unsigned kept = 0u;  // a bit an output of this lane
  for (int j = 0; j < keep; ++j) {
    float best;
    const int g = wave_argmax(score, lane, &best);
#pragma unroll
    for (int i = 0; i < PL; ++i) {
      if (lane + 64 * i == g) score[i] = -INFINITY;
      if (group[i] == g) kept |= 1u << i;
    }
  }
#pragma unroll
  for (int i = 0; i < PL; ++i)
    if (!(kept >> i & 1u)) c[i] = -INFINITY;
}

template <int PL>
__device__ __forceinline__ void route_outputs(const float* __restrict__ zr, const RouteArgs& a, int top, int* __restrict__ idx,
                                            float* __restrict__ weight, int lane) {
  const int n_out = a.n_out;
  float v[PL], c[PL];
  float m = -INFINITY;
#pragma unroll
  for (int i = 0; i < PL; ++i) {
    const int e = lane + 64 * i;
    v[i] = e < n_out ? zr[e] : -INFINITY;
    m = fmaxf(m, v[i]);
  }
  if (a.sigmoid) {
#pragma unroll
    for (int i = 0; i < PL; ++i) v[i] = 1.0f / (1.0f + expf(-v[i]));
  } else {
    m = wave_max(m);
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < PL; ++i) {
      v[i] = lane + 64 * i < n_out ? expf(v[i] - m) : 0.f;
      sum += v[i];
    }
    const float inv = 1.0f / wave_sum(sum);
#pragma unroll
    for (int i = 0; i < PL; ++i) v[i] *= inv;
  }
#pragma unroll
  for (int i = 0; i < PL; ++i) {
    const int e = lane + 64 * i;
    c[i] = e < n_out ? (a.correction ? v[i] + a.correction[e] : v[i]) : -INFINITY;
  }
  if (a.groups > 1) limit_groups(c, n_out, a.groups, a.keep, lane);
  float mine[PL];  // pick j's weight, kept by lane j % 64 until the picks' sum is known
#pragma unroll
  for (int i = 0; i < PL; ++i) mine[i] = 0.f;
  float total = 0.f;
  for (int j = 0; j < top; ++j) {
    float best;
    const int e = wave_argmax(c, lane, &best);
    float w = 0.f;
#pragma unroll
    for (int i = 0; i < PL; ++i)
      if (lane + 64 * i == e) {
        idx[j] = e, w = v[i];
        c[i] = -INFINITY;  // picked
      }
    w = wave_sum(w);  // (one lane holds it)
    total += w;
#pragma unroll
    for (int i = 0; i < PL; ++i)
      if (lane == (j & 63) && i == (j >> 6)) mine[i] = w;
  }
  const float factor = a.renorm ? a.mult / (total + 1e-20f) : a.mult;
#pragma unroll
  for (int i = 0; i < PL; ++i)
    if (lane + 64 * i < top) weight[lane + 64 * i] = mine[i] * factor;
}

// (up to 64 outputs: one a lane)
__device__ __forceinline__ void route_token(const float* __restrict__ zr, const RouteArgs& a, int top, int* __restrict__ idx,
                                            float* __restrict__ weight, int lane) {
  if (a.n_out <= 64) route_outputs<1>(zr, a, top, idx, weight, lane);
  else route_outputs<ROUTER_PER_LANE>(zr, a, top, idx, weight, lane);
}

__global__ __launch_bounds__(256) void router_choice_kernel(RouteArgs a, int n_tokens, int top, int* __restrict__ idx,
                                                            float* __restrict__ weight) {
  const int lane = threadIdx.x & 63, t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t >= n_tokens) return;  // whole waves leave; no barrier follows
  route_token(a.z + (size_t)t * a.ldz, a, top, idx + (size_t)t * top, weight + (size_t)t * top, lane);
}

// For a step of few tokens, where one product gave [router | gate | up] as float rows: a block a
// token, its first wave chooses the experts, all of it makes act = silu(gate) * up.
template <typename T>
__global__ __launch_bounds__(256) void route_and_gate_kernel(RouteArgs a, int top, int F, int* __restrict__ idx,
                                                             float* __restrict__ weight, T* __restrict__ act, int ldo) {
  const int t = blockIdx.x, lane = threadIdx.x & 63, n_out = a.n_out;
  const float* row = a.z + (size_t)t * a.ldz;
  if (threadIdx.x < 64) route_token(row, a, top, idx + (size_t)t * top, weight + (size_t)t * top, lane);
  for (int f = threadIdx.x; f < F; f += 256) act[(size_t)t * ldo + f] = from_f32<T>(silu_f(row[n_out + f]) * row[n_out + F + f]);
}

// GELU: the gate passes the tanh form of gelu instead of silu
template <typename T, bool GELU>
__global__ __launch_bounds__(256) void silu_mul_kernel(const T* __restrict__ gu, int ld, T* __restrict__ out, int ldo,
                                                       int n_rows, int F) {
  const int f = blockIdx.y * 256 + threadIdx.x, r = blockIdx.x;
  if (f >= F) return;
  const T* row = gu + (size_t)r * ld;
  const float z = to_f32(row[f]);
  out[(size_t)r * ldo + f] = from_f32<T>((GELU ? gelu_tanh(z) : silu_f(z)) * to_f32(row[F + f]));
}

// ROWS dot products of one vector b with ROWS rows a[r] over a lane's share of K, all loads of a step on
// their way at once: 16 bytes a lane and load where K and the rows allow (VEC), a value a lane otherwise.
template <typename T, bool VEC, int ROWS>
__device__ __forceinline__ void lane_dots(const T* const* __restrict__ a, const T* __restrict__ b, int K, int lane, float* s) {
#pragma unroll
  for (int r = 0; r < ROWS; ++r) s[r] = 0.f;
  if (VEC) {
    constexpr int W = 16 / sizeof(T);
    for (int k = lane * W; k < K; k += 64 * W) {
      u32x4_t av[ROWS];
      const u32x4_t bv = *(const u32x4_t*)(b + k);
#pragma unroll
      for (int r = 0; r < ROWS; ++r) av[r] = *(const u32x4_t*)(a[r] + k);
      const T* bp = (const T*)&bv;
#pragma unroll
      for (int r = 0; r < ROWS; ++r) {
        const T* ap = (const T*)&av[r];
#pragma unroll
        for (int i = 0; i < W; ++i) s[r] += to_f32(ap[i]) * to_f32(bp[i]);
      }
    }
  } else {
    for (int k = lane; k < K; k += 64) {
      const float bv = to_f32(b[k]);
#pragma unroll
      for (int r = 0; r < ROWS; ++r) s[r] += to_f32(a[r][k]) * bv;
    }
  }
}

#define ROUTED_MOST 64  // picks a token that a block chooses itself

// Block (token x pick, 16 features): a wave four features at once (eight rows of weights in
// flight), lanes along the width.  ROUTED: the block's first wave chooses the token's experts from the
// router's outputs; the block of the first pick and features leaves the choice for the kernel behind.
template <typename T, bool VEC, bool ROUTED>
__global__ __launch_bounds__(256) void expert_rows_up_kernel(const T* __restrict__ x, int ldx,
                                                             const T* __restrict__ w_gate, const T* __restrict__ w_up,
                                                             int* __restrict__ idx, float* __restrict__ weight, int n_experts,
                                                             int top, int F, int width, T* __restrict__ act, ExpertAct fn,
                                                             RouteArgs route) {
  __shared__ int s_idx[ROUTED ? ROUTED_MOST : 1];
  __shared__ float s_weight[ROUTED ? ROUTED_MOST : 1];
  const int item = blockIdx.x, t = item / top;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  int e;
  float wt;
  if constexpr (ROUTED) {
    if (wave == 0)
      route_token(route.z + (size_t)t * route.ldz, route, top, s_idx, s_weight, lane);
    __syncthreads();
    const int j = item - t * top;
    if (j == 0 && blockIdx.y == 0 && (int)threadIdx.x < top)
      idx[(size_t)t * top + threadIdx.x] = s_idx[threadIdx.x], weight[(size_t)t * top + threadIdx.x] = s_weight[threadIdx.x];
    e = s_idx[j], wt = s_weight[j];
  } else {
    e = idx[item], wt = weight[item];
  }
  if (e >= n_experts) return;  // an identity expert: nothing to compute
  const int f0 = blockIdx.y * 16 + wave * 4;
  if (f0 >= F) return;  // (no barrier from here on)
  const T* rows[8];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const size_t f = (size_t)e * F + min(f0 + r, F - 1);
    rows[r] = w_gate + f * width, rows[4 + r] = w_up + f * width;
  }
  float s[8];
  lane_dots<T, VEC, 8>(rows, x + (size_t)t * ldx, width, lane, s);
#pragma unroll
  for (int r = 0; r < 8; ++r) s[r] = wave_sum(s[r]);
  if (lane < 4 && f0 + lane < F) {
    float g = s[0], u = s[4];
#pragma unroll
    for (int r = 1; r < 4; ++r)
      if (lane == r) g = s[r], u = s[4 + r];
    act[(size_t)item * F + f0 + lane] = from_f32<T>(wt * expert_act(fn, g, u));
  }
}

// The layer behind's norm of the rows that the experts' sum completes, where that norm needs nothing but
// the element: out = tanh(alpha y) w + b (out null: none).
struct NextNorm {
  const float* alpha;
  const float* w;
  const float* b;
  void* out;  // [tokens, width] of the compute dtype
};

// Block (token, 16 / PW columns): a wave four output columns at once, lanes along the features; PW waves
// share the token's picks (every PW-th each) and are summed in their order.
template <typename T, bool VEC, int PW>
__global__ __launch_bounds__(256) void expert_rows_down_kernel(const T* __restrict__ act, const T* __restrict__ w_down,
                                                               const int* __restrict__ idx,
                                                               const float* __restrict__ weight,
                                                               const T* __restrict__ x, int ldx, int n_experts, int top,
                                                               int F, int width, float* __restrict__ y, int ldy,
                                                               int accumulate, NextNorm next) {
  __shared__ float part[4][8];
  const int t = blockIdx.x;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, pw = wave % PW;
  const int n0 = blockIdx.y * (16 / PW) + wave / PW * 4;
  float tot[4] = {0.f, 0.f, 0.f, 0.f}, same = 0.f;
  for (int j = pw; j < top; j += PW) {
    const int e = idx[(size_t)t * top + j];
    if (e >= n_experts) {
      same += weight[(size_t)t * top + j];
      continue;
    }
    const T* rows[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) rows[r] = w_down + ((size_t)e * width + min(n0 + r, width - 1)) * F;
    float s[4];
    lane_dots<T, VEC, 4>(rows, act + ((size_t)t * top + j) * F, F, lane, s);
#pragma unroll
    for (int r = 0; r < 4; ++r) tot[r] += s[r];
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) tot[r] = wave_sum(tot[r]);
  if (PW > 1) {
    if (lane == 0) part[wave][0] = tot[0], part[wave][1] = tot[1], part[wave][2] = tot[2], part[wave][3] = tot[3], part[wave][4] = same;
    __syncthreads();
  }
  if (pw != 0 || lane >= 4 || n0 + lane >= width) return;
  float v = tot[0];
#pragma unroll
  for (int r = 1; r < 4; ++r)
    if (lane == r) v = tot[r];
#pragma unroll
  for (int i = 1; i < PW; ++i) v += part[wave + i][lane], same += part[wave + i][4];
  v += same * to_f32(x[(size_t)t * ldx + n0 + lane]);
  float* o = y + (size_t)t * ldy + n0 + lane;
  if (accumulate) v = *o + v;
  *o = v;
  if (next.out) ((T*)next.out)[(size_t)t * width + n0 + lane] = from_f32<T>(tanhf(*next.alpha * v) * next.w[n0 + lane] + next.b[n0 + lane]);
}

// ---------------------------------------------------------------------------
// many tokens: picks sorted by expert, a tile of picks a block

#define TILE_PICKS 64        // picks a tile of the 32-bit kernels
#define TILE_PICKS_LEAST 32  // the smallest tile of the bfloat16 kernels

// One block.  tiles: (expert, first place in `order`, picks) each, up to `tile_picks` picks a tile.
__global__ __launch_bounds__(1024) void expert_sort_kernel(const int* __restrict__ idx, int n_items, int n_experts,
                                                           int tile_picks, int* __restrict__ order, int* __restrict__ tiles,
                                                           int* __restrict__ n_tiles) {
  extern __shared__ int lds_i[];
  int* counts = lds_i;
  int* cursor = lds_i + n_experts;
  int* first_tile = cursor + n_experts;
  for (int e = threadIdx.x; e < n_experts; e += 1024) counts[e] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < n_items; i += 1024) {
    const int e = idx[i];
    if (e < n_experts) atomicAdd(&counts[e], 1);
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    int at = 0, nt = 0;
    for (int e = 0; e < n_experts; ++e) {
      cursor[e] = at, first_tile[e] = nt;
      at += counts[e], nt += (counts[e] + tile_picks - 1) / tile_picks;
    }
    *n_tiles = nt;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < n_experts; e += 1024) {
    int* tile = tiles + 3 * first_tile[e];
    for (int r0 = 0; r0 < counts[e]; r0 += tile_picks, tile += 3)
      tile[0] = e, tile[1] = cursor[e] + r0, tile[2] = min(tile_picks, counts[e] - r0);
  }
  __syncthreads();  // (the cursors move from here on)
  for (int i = threadIdx.x; i < n_items; i += 1024) {
    const int e = idx[i];
    if (e < n_experts) order[atomicAdd(&cursor[e], 1)] = i;  // (any order within an expert: a pick's row is computed by itself)
  }
}

// A lane's share of a 16 x 16 product's operands: row (or column) lane % 16, KL values of k from
// KL * (lane / 16) on; the sums land as rows 4 (lane / 16) + i, column lane % 16.
template <typename T>
struct Frag;
template <>
struct Frag<bf16> {
  typedef bf16x8_t V;
  static constexpr int KL = 8;
  // (a lane beyond K brings zeros: the matrix instruction takes every lane's registers, whatever
  // the lanes' state, so the product itself must not stand under a condition)
  static __device__ __forceinline__ V load(const bf16* p, bool inside) {
    u32x4_t bits = {0u, 0u, 0u, 0u};
    if (inside) bits = *(const u32x4_t*)p;
    return __builtin_bit_cast(bf16x8_t, bits);
  }
  static __device__ __forceinline__ f32x4_t mma(V a, V b, f32x4_t c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
  }
};
template <>
struct Frag<float> {
  typedef f32x4_t V;
  static constexpr int KL = 4;
  static __device__ __forceinline__ V load(const float* p, bool inside) {
    f32x4_t v = {0.f, 0.f, 0.f, 0.f};
    if (inside) v = *(const f32x4_t*)p;
    return v;
  }
  static __device__ __forceinline__ f32x4_t mma(V a, V b, f32x4_t c) {
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, c, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, c, 0, 0, 0);
  }
};

// Block (tile, 64 CF features): a wave all of the tile's picks (four groups of 16) x 16 CF features
// of gate and of up, operands straight from memory; a weight fragment meets up to four fragments
// of rows.  CF = 4 where the tiles alone fill the GPU, 1 where they are few (a decode step of some
// dozen tokens), so that the blocks are four times as many.  act[pick, f] = weight * silu(gate) * up.
template <typename T, int CF>
__global__ __launch_bounds__(256) void expert_tiles_up_kernel(const T* __restrict__ x, int ldx, const T* __restrict__ w_gate,
                                                              const T* __restrict__ w_up, const int* __restrict__ order,
                                                              const int* __restrict__ tiles, const int* __restrict__ n_tiles,
                                                              const float* __restrict__ weight, int top, int F, int width,
                                                              T* __restrict__ act, ExpertAct fn) {
  typedef Frag<T> Fr;
  if ((int)blockIdx.x >= *n_tiles) return;
  const int e = tiles[3 * blockIdx.x], first = tiles[3 * blockIdx.x + 1], count = tiles[3 * blockIdx.x + 2];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4, r = lane & 15;
  const int f0 = (blockIdx.y * 4 + wave) * 16 * CF;
  if (f0 >= F) return;  // (no barrier in this kernel)
  const int groups = (count + 15) / 16;
  const T* xrow[4];
#pragma unroll
  for (int rg = 0; rg < 4; ++rg) xrow[rg] = x + (size_t)(order[first + min(16 * rg + r, count - 1)] / top) * ldx;
  const T* grow[CF];
  const T* urow[CF];
#pragma unroll
  for (int c = 0; c < CF; ++c) {
    const size_t f = (size_t)e * F + min(f0 + 16 * c + r, F - 1);
    grow[c] = w_gate + f * width, urow[c] = w_up + f * width;
  }
  f32x4_t ag[4][CF], au[4][CF];
#pragma unroll
  for (int rg = 0; rg < 4; ++rg)
#pragma unroll
    for (int c = 0; c < CF; ++c) ag[rg][c] = au[rg][c] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  // two sets of operands by turns: the next step's loads are on their way during this step's products
  // (the width is a multiple of KL: a lane's values are all inside or all outside)
  typename Fr::V a[2][4], bg[2][CF], bu[2][CF];
  const int step = 4 * Fr::KL;
#define LOAD_SET(S, K0)                                                                                 \
  do {                                                                                                  \
    const int k_ = (K0) + Fr::KL * g;                                                                   \
    const bool in_ = k_ < width;                                                                        \
    _Pragma("unroll") for (int rg = 0; rg < 4; ++rg) a[S][rg] = Fr::load(xrow[rg] + k_, in_);           \
    _Pragma("unroll") for (int c = 0; c < CF; ++c) bg[S][c] = Fr::load(grow[c] + k_, in_), bu[S][c] = Fr::load(urow[c] + k_, in_); \
  } while (0)
#define MMA_SET(S)                                                                                      \
  do {                                                                                                  \
    _Pragma("unroll") for (int rg = 0; rg < 4; ++rg) {                                                  \
      if (rg < groups) { /* (the same for every lane of the block) */                                   \
        _Pragma("unroll") for (int c = 0; c < CF; ++c) {                                                 \
          ag[rg][c] = Fr::mma(a[S][rg], bg[S][c], ag[rg][c]);                                           \
          au[rg][c] = Fr::mma(a[S][rg], bu[S][c], au[rg][c]);                                           \
        }                                                                                               \
      }                                                                                                 \
    }                                                                                                   \
  } while (0)
  LOAD_SET(0, 0);
  for (int k0 = 0; k0 < width; k0 += 2 * step) {
    LOAD_SET(1, k0 + step);  // (beyond the width: zeros, and nothing is read)
    MMA_SET(0);
    LOAD_SET(0, k0 + 2 * step);
    MMA_SET(1);
  }
#undef LOAD_SET
#undef MMA_SET
#pragma unroll
  for (int rg = 0; rg < 4; ++rg)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int ri = 16 * rg + 4 * g + i;
      if (ri >= count) continue;
      const int it = order[first + ri];
      const float wt = weight[it];
#pragma unroll
      for (int c = 0; c < CF; ++c) {
        const int f = f0 + 16 * c + r;
        if (f < F) act[(size_t)it * F + f] = from_f32<T>(wt * expert_act(fn, ag[rg][c][i], au[rg][c][i]));
      }
    }
}

// Block (tile, 64 CF columns): out[pick, n] = sum_f act[pick, f] w_down[e, n, f], laid out as above.
template <typename T, int CF>
__global__ __launch_bounds__(256) void expert_tiles_down_kernel(const T* __restrict__ act, const T* __restrict__ w_down,
                                                                const int* __restrict__ order, const int* __restrict__ tiles,
                                                                const int* __restrict__ n_tiles, int F, int width,
                                                                float* __restrict__ out) {
  typedef Frag<T> Fr;
  if ((int)blockIdx.x >= *n_tiles) return;
  const int e = tiles[3 * blockIdx.x], first = tiles[3 * blockIdx.x + 1], count = tiles[3 * blockIdx.x + 2];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4, r = lane & 15;
  const int n0 = (blockIdx.y * 4 + wave) * 16 * CF;
  if (n0 >= width) return;
  const int groups = (count + 15) / 16;
  const T* arow[4];
#pragma unroll
  for (int rg = 0; rg < 4; ++rg) arow[rg] = act + (size_t)order[first + min(16 * rg + r, count - 1)] * F;
  const T* drow[CF];
#pragma unroll
  for (int c = 0; c < CF; ++c) drow[c] = w_down + ((size_t)e * width + min(n0 + 16 * c + r, width - 1)) * F;
  f32x4_t acc[4][CF];
#pragma unroll
  for (int rg = 0; rg < 4; ++rg)
#pragma unroll
    for (int c = 0; c < CF; ++c) acc[rg][c] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  typename Fr::V a[2][4], b[2][CF];
  const int step = 4 * Fr::KL;
#define LOAD_SET(S, K0)                                                                        \
  do {                                                                                         \
    const int k_ = (K0) + Fr::KL * g;                                                          \
    const bool in_ = k_ < F;                                                                   \
    _Pragma("unroll") for (int rg = 0; rg < 4; ++rg) a[S][rg] = Fr::load(arow[rg] + k_, in_);  \
    _Pragma("unroll") for (int c = 0; c < CF; ++c) b[S][c] = Fr::load(drow[c] + k_, in_);       \
  } while (0)
#define MMA_SET(S)                                                                             \
  do {                                                                                         \
    _Pragma("unroll") for (int rg = 0; rg < 4; ++rg) {                                         \
      if (rg < groups) {                                                                       \
        _Pragma("unroll") for (int c = 0; c < CF; ++c) acc[rg][c] = Fr::mma(a[S][rg], b[S][c], acc[rg][c]); \
      }                                                                                        \
    }                                                                                          \
  } while (0)
  LOAD_SET(0, 0);
  for (int k0 = 0; k0 < F; k0 += 2 * step) {
    LOAD_SET(1, k0 + step);
    MMA_SET(0);
    LOAD_SET(0, k0 + 2 * step);
    MMA_SET(1);
  }
#undef LOAD_SET
#undef MMA_SET
#pragma unroll
  for (int rg = 0; rg < 4; ++rg)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int ri = 16 * rg + 4 * g + i;
      if (ri >= count) continue;
      const size_t it = order[first + ri];
#pragma unroll
      for (int c = 0; c < CF; ++c) {
        const int n = n0 + 16 * c + r;
        if (n < width) out[it * width + n] = acc[rg][c][i];
      }
    }
}

// The bfloat16 kernels for many tokens: both products as tiles through LDS.  A block takes one tile of
// picks (BM = 32 WM TM of one expert, gathered through the sorted list) and BN = 64 WN rows of that
// expert's weights; WM x WN waves, each 32 TM picks x 64 weight rows on v_mfma_f32_32x32x16_bf16, the
// weights as the instruction's rows, so that a lane ends up with four neighbouring outputs of a pick.
// UP: a wave's 64 weight rows are the gate's and the up projection's rows of the same 32 features, so
// the activation is the wave's own; down: 64 output columns.  Two k-blocks of 64 columns lie in LDS, two
// more are on their way in registers.  Blocks go to the eight dies in turn; the (tile, weight rows)
// pairs are put in panels of PANEL tiles, weight rows after weight rows inside a panel, and that
// sequence is cut into eight runs, one a die: the tiles of an expert meet its weights in one L2.
// The grid is as large as the tiles could be at most; blocks beyond those that there are leave at once.
#define XK 64              // columns a k-block
#define X_ZERO make_uint4(0u, 0u, 0u, 0u)  // a constant: a select against a variable would go through scratch memory
#define X_STRIDE (XK + 8)  // LDS row stride: 16-byte reads of neighbouring rows on distinct banks
template <int WM, int WN, int TM, bool UP>
__global__ __launch_bounds__(64 * WM * WN, 2) void expert_gemm_kernel(const uint16_t* __restrict__ x, int ldx,
                                                                   const uint16_t* __restrict__ w_a,
                                                                   const uint16_t* __restrict__ w_b,
                                                                   const int* __restrict__ order, const int* __restrict__ tiles,
                                                                   const int* __restrict__ n_tiles,
                                                                   const float* __restrict__ weight, int top, int N, int K,
                                                                   void* __restrict__ out, ExpertAct fn) {
  constexpr int BM = WM * TM * 32, BN = WN * 64, THREADS = 64 * WM * WN, ROW_STEP = THREADS / 8;
  constexpr int PA = BM / ROW_STEP, PB = BN / ROW_STEP, PANEL = BM >= 128 ? 4 : 8;
  __shared__ __attribute__((aligned(16))) uint16_t smem[2 * (BM + BN) * X_STRIDE];
  const int nt = *n_tiles, columns = UP ? BN / 2 : BN, nb = (N + columns - 1) / columns;
  const int total = nt * nb, run = (total + N_DIES - 1) / N_DIES, local = blockIdx.x / N_DIES;
  const int at = (int)(blockIdx.x % N_DIES) * run + local;
  if (local >= run || at >= total) return;
  const int panel = at / (PANEL * nb), rem = at - panel * PANEL * nb, tall = min(PANEL, nt - panel * PANEL);
  const int tile = panel * PANEL + rem % tall, fb = rem / tall;
  const int e = tiles[3 * tile], first = tiles[3 * tile + 1], count = tiles[3 * tile + 2];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, wm = wave / WN, wn = wave % WN;

  // a thread moves PA pieces of 16 bytes of the picks' rows and PB of the weights' per k-block: piece i
  // is row tid / 8 + ROW_STEP i, columns 8 (tid % 8) ..; rows beyond the tile repeat rows inside it
  const int kc = (tid & 7) * 8;
  int pa[PA], pb[PB];  // (element offsets of 32 bits: registers are scarce here)
  const uint16_t* wa = w_a + (size_t)e * N * K;
  const uint16_t* wb = UP ? w_b + (size_t)e * N * K : wa;
#pragma unroll
  for (int i = 0; i < PA; ++i) {
    const int r = (tid >> 3) + ROW_STEP * i, item = order[first + (r < count ? r : r % count)];
    pa[i] = (UP ? item / top : item) * ldx + kc;
  }
#pragma unroll
  for (int i = 0; i < PB; ++i) {
    const int c = (tid >> 3) + ROW_STEP * i;
    const int f = UP ? fb * columns + (c >> 6) * 32 + (c & 31) : fb * columns + c;
    pb[i] = (f < N ? f : f % N) * K + kc;
  }
  uint4 ra[2][PA], rb[2][PB];
  auto load = [&](uint4 (&xa)[PA], uint4 (&xb)[PB], int k0) {
    const int kk = k0 + kc < K ? k0 : -kc;  // (a piece beyond K: the row's first columns, zeroed on their way to LDS)
#pragma unroll
    for (int i = 0; i < PA; ++i) xa[i] = *(const uint4*)(x + (pa[i] + kk));
    // (32 rows of the gate, 32 of the up projection by turns: which of the two a piece belongs to is known)
#pragma unroll
    for (int i = 0; i < PB; ++i) xb[i] = *(const uint4*)(((ROW_STEP * i) & 32 ? wb : wa) + (pb[i] + kk));
  };
  static_assert(!UP || ROW_STEP == 32 || ROW_STEP == 16, "a thread's pieces lie in one of the two matrices each");
  const int lds_at = (tid >> 3) * X_STRIDE + kc;
  auto store = [&](int stage, const uint4 (&xa)[PA], const uint4 (&xb)[PB], int k0) {
    const bool in = k0 + kc < K;
    uint16_t* a = smem + stage * (BM + BN) * X_STRIDE + lds_at;
    uint16_t* b = a + BM * X_STRIDE;
#pragma unroll
    for (int i = 0; i < PA; ++i) *(uint4*)(a + i * ROW_STEP * X_STRIDE) = in ? xa[i] : X_ZERO;
#pragma unroll
    for (int i = 0; i < PB; ++i) *(uint4*)(b + i * ROW_STEP * X_STRIDE) = in ? xb[i] : X_ZERO;
  };
  f32x16_t acc[TM][2];
#pragma unroll
  for (int i = 0; i < TM; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[i][j][r] = 0.f;
  auto multiply = [&](int stage) {
    const uint16_t* a = smem + stage * (BM + BN) * X_STRIDE + (wm * TM * 32 + (lane & 31)) * X_STRIDE + (lane >> 5) * 8;
    const uint16_t* b = smem + (stage * (BM + BN) + BM) * X_STRIDE + (wn * 64 + (lane & 31)) * X_STRIDE + (lane >> 5) * 8;
#pragma unroll
    for (int ks = 0; ks < XK; ks += 16) {
      bf16x8_t av[TM], bv[2];
#pragma unroll
      for (int i = 0; i < TM; ++i) av[i] = *(const bf16x8_t*)(a + i * 32 * X_STRIDE + ks);
#pragma unroll
      for (int j = 0; j < 2; ++j) bv[j] = *(const bf16x8_t*)(b + j * 32 * X_STRIDE + ks);
#pragma unroll
      for (int i = 0; i < TM; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(bv[j], av[i], acc[i][j], 0, 0, 0);
    }
  };
  const int blocks = (K + XK - 1) / XK, last = (blocks - 1) * XK;
  load(ra[0], rb[0], 0);
  load(ra[1], rb[1], min(XK, last));
  store(0, ra[0], rb[0], 0);
  __syncthreads();
  for (int kb = 0; kb < blocks; kb += 2) {
    load(ra[0], rb[0], min((kb + 2) * XK, last));
    __builtin_amdgcn_sched_barrier(0);  // (the loads go out ahead of the arithmetic)
    multiply(0);
    store(1, ra[1], rb[1], min((kb + 1) * XK, last));
    __syncthreads();
    if (kb + 1 >= blocks) break;
    load(ra[1], rb[1], min((kb + 3) * XK, last));
    __builtin_amdgcn_sched_barrier(0);
    multiply(1);
    store(0, ra[0], rb[0], min((kb + 2) * XK, last));
    __syncthreads();
  }
  // register r of a 32 x 32 tile: weight row 8 (r / 4) + 4 (lane / 32) + r % 4, pick lane % 32
#pragma unroll
  for (int i = 0; i < TM; ++i) {
    const int r = (wm * TM + i) * 32 + (lane & 31);
    if (r >= count) continue;
    const int item = order[first + r];
    if constexpr (UP) {
      const float wt = weight[item];
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        const int f = fb * columns + wn * 32 + 8 * g + 4 * (lane >> 5);
        if (f >= N) continue;  // (N is a multiple of eight: a piece of four is inside or outside)
        float v[4];
#pragma unroll
        for (int c = 0; c < 4; ++c) v[c] = wt * expert_act(fn, acc[i][0][4 * g + c], acc[i][1][4 * g + c]);
        *(uint2*)((uint16_t*)out + (size_t)item * N + f) = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
      }
    } else {
#pragma unroll
      for (int j = 0; j < 2; ++j)
#pragma unroll
        for (int g = 0; g < 4; ++g) {
          const int n = fb * columns + wn * 64 + 32 * j + 8 * g + 4 * (lane >> 5);
          if (n >= N) continue;
          *(float4*)((float*)out + (size_t)item * N + n) =
              make_float4(acc[i][j][4 * g], acc[i][j][4 * g + 1], acc[i][j][4 * g + 2], acc[i][j][4 * g + 3]);
        }
    }
  }
}

// Thread (token, column): a token's picks in their order, identity experts give weight * x.
template <typename T>
__global__ __launch_bounds__(256) void expert_combine_kernel(const float* __restrict__ out, const int* __restrict__ idx,
                                                             const float* __restrict__ weight, const T* __restrict__ x, int ldx,
                                                             int n_experts, int top, int width, float* __restrict__ y, int ldy,
                                                             int accumulate, NextNorm next) {
  const int n = blockIdx.y * 256 + threadIdx.x, t = blockIdx.x;
  if (n >= width) return;
  float s = 0.f, same = 0.f;
  for (int j = 0; j < top; ++j) {
    const size_t it = (size_t)t * top + j;
    if (idx[it] >= n_experts)
      same += weight[it];
    else
      s += out[it * width + n];
  }
  float v = s + same * to_f32(x[(size_t)t * ldx + n]);
  float* o = y + (size_t)t * ldy + n;
  if (accumulate) v = *o + v;
  *o = v;
  if (next.out) ((T*)next.out)[(size_t)t * width + n] = from_f32<T>(tanhf(*next.alpha * v) * next.w[n] + next.b[n]);
}

DEFINE_LAST_ERROR(mlxlm_last_error)

static int check_route(const char* who, const RouteArgs& a, int top) {
  if (!a.z || a.n_out <= 0 || top <= 0 || top > a.n_out || a.ldz < a.n_out)
    FAIL("%s: %d of %d outputs, rows of %d", who, top, a.n_out, a.ldz);
  if (a.n_out > 64 * ROUTER_PER_LANE) FAIL("%s: %d outputs, at most %d", who, a.n_out, 64 * ROUTER_PER_LANE);
  if (a.groups > 1 && (a.n_out % a.groups || a.keep <= 0 || a.keep > a.groups || top > a.keep * (a.n_out / a.groups)))
    FAIL("%s: %d picks of %d of %d groups of %d outputs", who, top, a.keep, a.groups, a.n_out);
  return 0;
}

// router_choice: a.z are the tokens' router outputs; idx, weight: [n_tokens, top].
extern "C" int router_choice(const RouteArgs* args, int n_tokens, int top, int* idx, float* weight, hipStream_t stream) {
  if (n_tokens <= 0) return 0;
  if (!args || !idx || !weight) FAIL("router_choice: null pointer");
  if (check_route("router_choice", *args, top)) return 1;
  hipLaunchKernelGGL(router_choice_kernel, dim3((n_tokens + 3) / 4), dim3(256), 0, stream, *args, n_tokens, top, idx, weight);
  CHECK_LAUNCH("router_choice");
  return 0;
}

// route_and_gate: a.z are rows [router outputs | F gate columns | F up columns].
extern "C" int route_and_gate(const RouteArgs* args, int n_tokens, int top, int F, int* idx, float* weight, void* act, int ldo,
                              int dtype, hipStream_t stream) {
  if (n_tokens <= 0) return 0;
  if (!args || !idx || !weight || !act) FAIL("route_and_gate: null pointer");
  if (check_route("route_and_gate", *args, top)) return 1;
  if (F <= 0 || args->ldz < args->n_out + 2 * F || ldo < F)
    FAIL("route_and_gate: %d outputs and 2 x %d columns in rows of %d", args->n_out, F, args->ldz);
  if (dtype != DT_F32 && dtype != DT_BF16) FAIL("route_and_gate: unknown dtype code %d", dtype);
  if (dtype == DT_F32)
    hipLaunchKernelGGL(route_and_gate_kernel<float>, dim3(n_tokens), dim3(256), 0, stream, *args, top, F, idx, weight,
                       (float*)act, ldo);
  else
    hipLaunchKernelGGL(route_and_gate_kernel<bf16>, dim3(n_tokens), dim3(256), 0, stream, *args, top, F, idx, weight,
                       (bf16*)act, ldo);
  CHECK_LAUNCH("route_and_gate");
  return 0;
}

// act_mul: out = act(gate) * up for rows [gate | up]; `activation` 0: silu, 1: the tanh form of gelu.
static int act_mul_launch(const void* gu, int ld, void* out, int ldo, int n_rows, int F, int dtype, int activation,
                          hipStream_t stream) {
  if (n_rows <= 0 || F <= 0) return 0;
  if (activation != 0 && activation != 1) FAIL("act_mul: unknown activation code %d", activation);
  if (!gu || !out) FAIL("silu_mul: null pointer");
  if (ld < 2 * F || ldo < F) FAIL("silu_mul: rows of %d for 2 x %d, output rows of %d", ld, F, ldo);
  if (dtype != DT_F32 && dtype != DT_BF16) FAIL("silu_mul: unknown dtype code %d", dtype);
  dim3 grid(n_rows, (F + 255) / 256), block(256);
  if (dtype == DT_F32) {
    if (activation)
      hipLaunchKernelGGL((silu_mul_kernel<float, true>), grid, block, 0, stream, (const float*)gu, ld, (float*)out, ldo, n_rows, F);
    else
      hipLaunchKernelGGL((silu_mul_kernel<float, false>), grid, block, 0, stream, (const float*)gu, ld, (float*)out, ldo, n_rows, F);
  } else {
    if (activation)
      hipLaunchKernelGGL((silu_mul_kernel<bf16, true>), grid, block, 0, stream, (const bf16*)gu, ld, (bf16*)out, ldo, n_rows, F);
    else
      hipLaunchKernelGGL((silu_mul_kernel<bf16, false>), grid, block, 0, stream, (const bf16*)gu, ld, (bf16*)out, ldo, n_rows, F);
  }
  CHECK_LAUNCH("silu_mul");
  return 0;
}

extern "C" int silu_mul(const void* gu, int ld, void* out, int ldo, int n_rows, int F, int dtype, hipStream_t stream) {
  return act_mul_launch(gu, ld, out, ldo, n_rows, F, dtype, 0, stream);
}

extern "C" int act_mul(const void* gu, int ld, void* out, int ldo, int n_rows, int F, int dtype, int activation,
                       hipStream_t stream) {
  return act_mul_launch(gu, ld, out, ldo, n_rows, F, dtype, activation, stream);
}

// act: [n_tokens * top, F] of the compute dtype; y: float rows.  `route` (or null): the choice is made
// here, from the router's outputs, into idx and weight.  `next` (or null): the norm of the new rows.
extern "C" int expert_rows(const void* x, int ldx, const void* w_gate, const void* w_up, const void* w_down,
                           int* idx, float* weight, int n_tokens, int n_experts, int top, int F, int width,
                           void* act, float* y, int ldy, int accumulate, int dtype, int act_kind, float act_limit,
                           const RouteArgs* route, const NextNorm* next, hipStream_t stream) {
  if (n_tokens <= 0) return 0;
  if (!x || !idx || !weight || !y || (n_experts > 0 && (!w_gate || !w_up || !w_down || !act)))
    FAIL("expert_rows: null pointer");
  if (top <= 0 || F <= 0 || width <= 0 || ldx < width || ldy < width) FAIL("expert_rows: sizes");
  if (dtype != DT_F32 && dtype != DT_BF16) FAIL("expert_rows: unknown dtype code %d", dtype);
  if (act_kind != EXPERT_SILU && act_kind != EXPERT_CLAMPED) FAIL("expert_rows: unknown activation code %d", act_kind);
  const ExpertAct fn = {act_kind, act_limit};
  if (route) {
    if (n_experts <= 0 || top > ROUTED_MOST) FAIL("expert_rows: %d picks of %d experts are not chosen here", top, n_experts);
    if (check_route("expert_rows", *route, top)) return 1;
  }
  const NextNorm nn = next ? *next : NextNorm{};
  if (next && (!nn.out || !nn.alpha || !nn.w || !nn.b || !accumulate)) FAIL("expert_rows: the next norm's pointers, or rows that are not complete here");
  const RouteArgs rt = route ? *route : RouteArgs{};
  const int feats = 16, per = dtype == DT_BF16 ? 8 : 4, pw = top >= 4 ? 4 : top >= 2 ? 2 : 1, cols = 16 / pw;
  const bool vec = F % per == 0 && width % per == 0 && ldx % per == 0 && !((uintptr_t)x & 15);
  dim3 block(256), up_grid(n_tokens * top, (F + feats - 1) / feats), down_grid(n_tokens, (width + cols - 1) / cols);
#define UP(T, VEC, ROUTED)                                                                                                  \
  hipLaunchKernelGGL((expert_rows_up_kernel<T, VEC, ROUTED>), up_grid, block, 0, stream, (const T*)x, ldx, (const T*)w_gate, \
                     (const T*)w_up, idx, weight, n_experts, top, F, width, (T*)act, fn, rt)
#define DOWN(T, VEC, PW)                                                                                                   \
  hipLaunchKernelGGL((expert_rows_down_kernel<T, VEC, PW>), down_grid, block, 0, stream, (const T*)act, (const T*)w_down,  \
                     idx, weight, (const T*)x, ldx, n_experts, top, F, width, y, ldy, accumulate, nn)
#define RUN(T, VEC)                         \
  do {                                      \
    if (n_experts > 0) {                    \
      if (route) UP(T, VEC, true);          \
      else UP(T, VEC, false);               \
    }                                       \
    if (pw == 4) DOWN(T, VEC, 4);           \
    else if (pw == 2) DOWN(T, VEC, 2);      \
    else DOWN(T, VEC, 1);                   \
  } while (0)
  if (dtype == DT_F32) {
    if (vec) RUN(float, true); else RUN(float, false);
  } else {
    if (vec) RUN(bf16, true); else RUN(bf16, false);
  }
#undef RUN
#undef UP
#undef DOWN
  CHECK_LAUNCH("expert_rows");
  return 0;
}

// The most tiles that n_items picks over n_experts experts can make.
extern "C" int expert_tiles_most(int n_items, int n_experts) {
  return (n_items + TILE_PICKS_LEAST - 1) / TILE_PICKS_LEAST + n_experts;
}

// 1 if expert_tiles takes these sizes (the operands are read 16 bytes a lane).
extern "C" int expert_tiles_takes(int F, int width, int dtype) {
  const int kl = dtype == DT_BF16 ? 8 : 4;
  return F > 0 && F % kl == 0 && width % kl == 0;
}

// order: [n_tokens * top] ints, tiles: [3 * expert_tiles_most] ints, n_tiles: one int, act: [n_tokens * top, F]
// of the compute dtype, out: [n_tokens * top, width] floats.  `next` (or null): the norm of the new rows.
extern "C" int expert_tiles(const void* x, int ldx, const void* w_gate, const void* w_up, const void* w_down, const int* idx,
                            const float* weight, int n_tokens, int n_experts, int top, int F, int width, int* order, int* tiles,
                            int* n_tiles, void* act, float* out, float* y, int ldy, int accumulate, int dtype,
                            int act_kind, float act_limit, const NextNorm* next, hipStream_t stream) {
  if (n_tokens <= 0) return 0;
  const NextNorm nn = next ? *next : NextNorm{};
  if (next && (!nn.out || !nn.alpha || !nn.w || !nn.b || !accumulate)) FAIL("expert_tiles: the next norm's pointers, or rows that are not complete here");
  if (!x || !idx || !weight || !y || !w_gate || !w_up || !w_down || !order || !tiles || !n_tiles || !act || !out)
    FAIL("expert_tiles: null pointer");
  if (n_experts <= 0 || top <= 0 || ldx < width || ldy < width) FAIL("expert_tiles: sizes");
  if (dtype != DT_F32 && dtype != DT_BF16) FAIL("expert_tiles: unknown dtype code %d", dtype);
  if (!expert_tiles_takes(F, width, dtype)) FAIL("expert_tiles: inner size %d and width %d must be multiples of %d", F, width, dtype == DT_BF16 ? 8 : 4);
  if (n_experts > 8192) FAIL("expert_tiles: %d experts are more than the sorting block's LDS holds", n_experts);
  if ((size_t)n_tokens * ldx >= (1u << 31) || (size_t)n_tokens * top * F >= (1u << 31) || (size_t)F * width >= (1u << 31))
    FAIL("expert_tiles: operands of 2^31 elements or more are not supported");
  if (ldx % (dtype == DT_BF16 ? 8 : 4) || ((uintptr_t)x & 15)) FAIL("expert_tiles: the rows of x must be 16-byte aligned");
  if (act_kind != EXPERT_SILU && act_kind != EXPERT_CLAMPED) FAIL("expert_tiles: unknown activation code %d", act_kind);
  const ExpertAct fn = {act_kind, act_limit};
  const int n_items = n_tokens * top;
  const dim3 block(256), sum_grid(n_tokens, (width + 255) / 256);
  // tiles of as many picks as an expert has on average: an expert's weights are then read about once
  const int each = n_items / n_experts;
  const int picks = dtype == DT_F32 ? TILE_PICKS : each >= 96 ? 128 : each >= 40 ? 64 : TILE_PICKS_LEAST;
  const int most = (n_items + picks - 1) / picks + n_experts;
  hipLaunchKernelGGL(expert_sort_kernel, dim3(1), dim3(1024), 3 * n_experts * sizeof(int), stream, idx, n_items, n_experts,
                     picks, order, tiles, n_tiles);
  if (dtype == DT_F32) {
    // (wide blocks where the tiles alone fill the GPU, narrow ones where they are few)
    const bool wide = (long)most * ((F + 255) / 256) >= 256;
    const int per = wide ? 256 : 64;
    const dim3 up_grid(most, (F + per - 1) / per), down_grid(most, (width + per - 1) / per);
#define RUN(CF)                                                                                                             \
  do {                                                                                                                      \
    hipLaunchKernelGGL((expert_tiles_up_kernel<float, CF>), up_grid, block, 0, stream, (const float*)x, ldx,                 \
                       (const float*)w_gate, (const float*)w_up, order, tiles, n_tiles, weight, top, F, width, (float*)act, fn); \
    hipLaunchKernelGGL((expert_tiles_down_kernel<float, CF>), down_grid, block, 0, stream, (const float*)act,                \
                       (const float*)w_down, order, tiles, n_tiles, F, width, out);                                         \
  } while (0)
    if (wide) RUN(4); else RUN(1);
#undef RUN
    hipLaunchKernelGGL(expert_combine_kernel<float>, sum_grid, block, 0, stream, out, idx, weight, (const float*)x, ldx, n_experts,
                       top, width, y, ldy, accumulate, nn);
  } else {
#define RUN(WM, WN, TM)                                                                                                     \
  do {                                                                                                                      \
    const long up_blocks = (long)most * ((F + 32 * WN - 1) / (32 * WN)), down_blocks = (long)most * ((width + 64 * WN - 1) / (64 * WN)); \
    hipLaunchKernelGGL((expert_gemm_kernel<WM, WN, TM, true>), dim3((unsigned)((up_blocks + 7) / 8 * 8)), dim3(64 * WM * WN), 0,  \
                       stream, (const uint16_t*)x, ldx, (const uint16_t*)w_gate, (const uint16_t*)w_up, order, tiles,         \
                       n_tiles, weight, top, F, width, act, fn);                                                            \
    hipLaunchKernelGGL((expert_gemm_kernel<WM, WN, TM, false>), dim3((unsigned)((down_blocks + 7) / 8 * 8)), dim3(64 * WM * WN), 0, \
                       stream, (const uint16_t*)act, F, (const uint16_t*)w_down, (const uint16_t*)nullptr, order, tiles,     \
                       n_tiles, weight, top, width, F, out, fn);                                                            \
  } while (0)
    if (picks == 128) RUN(2, 2, 2);
    else if (picks == 64) RUN(2, 2, 1);
    else RUN(1, 2, 1);
#undef RUN
    hipLaunchKernelGGL(expert_combine_kernel<bf16>, sum_grid, block, 0, stream, out, idx, weight, (const bf16*)x, ldx, n_experts,
                       top, width, y, ldy, accumulate, nn);
  }
  CHECK_LAUNCH("expert_tiles");
  return 0;
}
