// Dynamic Tanh, a norm that takes no mean and no variance:
//   y = tanh(alpha * x) * w + b        (alpha one number, w and b a value a column)
// over rows of the 32-bit stream, or over embedding rows on their way into the stream.
//
//   dynamic_tanh        rows of float x (all, or those listed in `rows`) to float or bfloat16
//   embed_dynamic_tanh  out[t] = tanh(alpha * scale * table[ids[t]]) * w + b, float
//   token_mix           the token shift behind such a norm, in one launch: h = the norm of a row,
//                       h' = the norm of the row before it in its sequence (zero ahead of the
//                       first; from the request's state row where it lies in an earlier step),
//                       and n_mix rows h + (h' - h) * mu_m for the products that each read a mix
//                       of their own.  Since the norm needs nothing but the element, h' is made
//                       again instead of kept.  The block of a request's first row of the step
//                       also leaves the normed last row in the state, after it has read the old one.
//
// Everything is 32-bit; only what goes to a bfloat16 output is rounded.  Also the native parts for
// the norm and for such an embedding (engine_parts.h).
#include "common.h"
#include "engine_parts.h"

struct TanhNorm {
  const float* alpha;  // one number, on the device
  const float* w;
  const float* b;
};

__device__ __forceinline__ float4 tanh_norm4(float4 x, float alpha, float4 w, float4 b) {
  return make_float4(tanhf(alpha * x.x) * w.x + b.x, tanhf(alpha * x.y) * w.y + b.y, tanhf(alpha * x.z) * w.z + b.z,
                     tanhf(alpha * x.w) * w.w + b.w);
}
__device__ __forceinline__ void store4(float* p, float4 v) { *(float4*)p = v; }
__device__ __forceinline__ void store4(bf16* p, float4 v) {
  *(uint2*)p = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w));
}

// A thread four columns of a row.
template <typename T>
__global__ __launch_bounds__(256) void dynamic_tanh_kernel(T* __restrict__ out, const float* __restrict__ x, int ldx,
                                                           const int* __restrict__ rows, TanhNorm n, int width) {
  const int r = blockIdx.x, k = (blockIdx.y * 256 + threadIdx.x) * 4;
  if (k >= width) return;
  const float4 v = *(const float4*)(x + (size_t)(rows ? rows[r] : r) * ldx + k);
  store4(out + (size_t)r * width + k, tanh_norm4(v, *n.alpha, *(const float4*)(n.w + k), *(const float4*)(n.b + k)));
}

template <typename T>
__global__ __launch_bounds__(256) void embed_dynamic_tanh_kernel(float* __restrict__ out, const T* __restrict__ table,
                                                                 const int* __restrict__ ids, float scale, TanhNorm n,
                                                                 int width) {
  const int r = blockIdx.x, k = (blockIdx.y * 256 + threadIdx.x) * 4;
  if (k >= width) return;
  const T* row = table + (size_t)ids[r] * width + k;
  const float4 v = make_float4(to_f32(row[0]) * scale, to_f32(row[1]) * scale, to_f32(row[2]) * scale, to_f32(row[3]) * scale);
  store4(out + (size_t)r * width + k, tanh_norm4(v, *n.alpha, *(const float4*)(n.w + k), *(const float4*)(n.b + k)));
}

struct TokenMixArgs {
  const float* x;  // [rows, ldx] the stream
  int ldx, n_rows, width;
  TanhNorm norm;
  const float* mu;  // [n_mix, width]
  int n_mix;
  void* out;  // [1 + n_mix][n_rows][width]: h, then the mixes
  float* state;  // a request's row: the last normed row of earlier steps, `width` floats at state_offset
  size_t state_stride, state_offset;
  const int* token_req;
  const int* seq_start;
  const int* seq_len;
  const int* slot_ids;
};

template <typename T>
__global__ __launch_bounds__(256) void token_mix_kernel(TokenMixArgs a) {
  const int r = blockIdx.x, k = (blockIdx.y * 256 + threadIdx.x) * 4;
  if (k >= a.width) return;
  const int req = a.token_req[r], start = a.seq_start[req];
  const bool first = r == start;
  const float* xr = a.x + (size_t)r * a.ldx + k;
  float* kept = a.state + (size_t)a.slot_ids[req] * a.state_stride + a.state_offset + k;  // (a row may start anywhere)
  const float4 w = *(const float4*)(a.norm.w + k), b = *(const float4*)(a.norm.b + k);
  const float alpha = *a.norm.alpha;
  const float4 xv = *(const float4*)xr;
  const float4 xp = *(const float4*)(first ? xr : xr - a.ldx);
  float4 hp;
  if (first)
    hp = make_float4(kept[0], kept[1], kept[2], kept[3]);
  else
    hp = tanh_norm4(xp, alpha, w, b);
  const float4 h = tanh_norm4(xv, alpha, w, b);
  const float4 d = make_float4(hp.x - h.x, hp.y - h.y, hp.z - h.z, hp.w - h.w);
  T* o = (T*)a.out + (size_t)r * a.width + k;
  const size_t plane = (size_t)a.n_rows * a.width;
  store4(o, h);
  for (int m = 0; m < a.n_mix; ++m) {
    const float4 mu = *(const float4*)(a.mu + (size_t)m * a.width + k);
    store4(o + (m + 1) * plane, make_float4(h.x + d.x * mu.x, h.y + d.y * mu.y, h.z + d.z * mu.z, h.w + d.w * mu.w));
  }
  if (first) {  // (this thread alone touches these four columns of the request's state)
    const int n = a.seq_len[req];
    const float4 last = n == 1 ? h : tanh_norm4(*(const float4*)(a.x + (size_t)(start + n - 1) * a.ldx + k), alpha, w, b);
    kept[0] = last.x, kept[1] = last.y, kept[2] = last.z, kept[3] = last.w;
  }
}

DEFINE_LAST_ERROR(mlxlm_last_error)

static int check_norm(const char* who, const TanhNorm& n, int width, int ldx) {
  if (!n.alpha || !n.w || !n.b) FAIL("%s: null pointer", who);
  if (width <= 0 || width % 4 || ldx % 4 || ldx < width) FAIL("%s: rows of %d floats, stride %d (multiples of 4)", who, width, ldx);
  if (((uintptr_t)n.w | (uintptr_t)n.b) & 15) FAIL("%s: weight and shift are 16-byte aligned", who);
  return 0;
}

extern "C" int dynamic_tanh(void* out, const float* x, int ldx, const int* rows, const float* alpha, const float* w,
                            const float* b, int n_rows, int width, int out_dtype, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  const TanhNorm n = {alpha, w, b};
  if (check_norm("dynamic_tanh", n, width, ldx)) return 1;
  if (!out || !x || (((uintptr_t)out | (uintptr_t)x) & 15)) FAIL("dynamic_tanh: 16-byte aligned rows");
  const dim3 grid(n_rows, (width / 4 + 255) / 256), block(256);
  if (out_dtype == DT_F32)
    hipLaunchKernelGGL(dynamic_tanh_kernel<float>, grid, block, 0, stream, (float*)out, x, ldx, rows, n, width);
  else if (out_dtype == DT_BF16)
    hipLaunchKernelGGL(dynamic_tanh_kernel<bf16>, grid, block, 0, stream, (bf16*)out, x, ldx, rows, n, width);
  else
    FAIL("dynamic_tanh: unknown dtype code %d", out_dtype);
  CHECK_LAUNCH("dynamic_tanh");
  return 0;
}

extern "C" int embed_dynamic_tanh(float* out, const void* table, int table_dtype, const int* ids, float scale,
                                  const float* alpha, const float* w, const float* b, int n_rows, int width,
                                  hipStream_t stream) {
  if (n_rows <= 0) return 0;
  const TanhNorm n = {alpha, w, b};
  if (check_norm("embed_dynamic_tanh", n, width, width)) return 1;
  if (!out || !table || !ids || ((uintptr_t)out & 15)) FAIL("embed_dynamic_tanh: null pointer, or rows not 16-byte aligned");
  const dim3 grid(n_rows, (width / 4 + 255) / 256), block(256);
  if (table_dtype == DT_F32)
    hipLaunchKernelGGL(embed_dynamic_tanh_kernel<float>, grid, block, 0, stream, out, (const float*)table, ids, scale, n, width);
  else if (table_dtype == DT_BF16)
    hipLaunchKernelGGL(embed_dynamic_tanh_kernel<bf16>, grid, block, 0, stream, out, (const bf16*)table, ids, scale, n, width);
  else
    FAIL("embed_dynamic_tanh: unknown dtype code %d", table_dtype);
  CHECK_LAUNCH("embed_dynamic_tanh");
  return 0;
}

extern "C" int token_mix(const TokenMixArgs* args, int out_dtype, hipStream_t stream) {
  const TokenMixArgs& a = *args;
  if (a.n_rows <= 0) return 0;
  if (check_norm("token_mix", a.norm, a.width, a.ldx)) return 1;
  if (!a.x || !a.mu || !a.out || !a.state || !a.token_req || !a.seq_start || !a.seq_len || !a.slot_ids)
    FAIL("token_mix: null pointer");
  if (((uintptr_t)a.x | (uintptr_t)a.mu | (uintptr_t)a.out) & 15) FAIL("token_mix: 16-byte aligned rows");
  if (a.n_mix < 1 || a.state_stride < a.state_offset + a.width) FAIL("token_mix: %d mixes, state rows of %zu floats", a.n_mix, a.state_stride);
  const dim3 grid(a.n_rows, (a.width / 4 + 255) / 256), block(256);
  if (out_dtype == DT_F32)
    hipLaunchKernelGGL(token_mix_kernel<float>, grid, block, 0, stream, a);
  else if (out_dtype == DT_BF16)
    hipLaunchKernelGGL(token_mix_kernel<bf16>, grid, block, 0, stream, a);
  else
    FAIL("token_mix: unknown dtype code %d", out_dtype);
  CHECK_LAUNCH("token_mix");
  return 0;
}

// ---------------------------------------------------------------------------
// the parts

static const EngHost* host = nullptr;

struct DynamicTanh : Norm {
  int width;
  TanhNorm n;
  DynamicTanh(int w, const TanhNorm& t) : width(w), n(t) {}
  int forward(EngCtx* ctx, const EngMat& x, const int* rows, int n_rows, bool, const EngWeight*, bool, EngValue* out) override {
    if (x.cols != width || x.dtype != DT_F32) return host->fail("dynamic tanh: float32 rows of width %d", width);
    *out = EngValue{};
    if (host->take(ctx, rows ? n_rows : x.rows, width, ctx->dtype, &out->m)) return 1;
    if (dynamic_tanh(out->m.p, (const float*)x.p, x.ld, rows, n.alpha, n.w, n.b, out->m.rows, width, ctx->dtype, ctx->stream))
      return host->fail("%s", g_err);
    host->launched(ctx);
    return 0;
  }
};

struct NormedTokens : Embedding {
  const void* table;
  int width, dtype;
  float scale;
  TanhNorm n;
  int forward(EngCtx* ctx, const EngMat& out, const EngMat& add_table, const int*) override {
    if (add_table.p) return host->fail("a normed embedding takes no position table");
    if (out.cols != width || out.dtype != DT_F32 || out.ld != width) return host->fail("embedding: out must be float32 [tokens, %d]", width);
    if (embed_dynamic_tanh((float*)out.p, table, dtype, ctx->token_ids, scale, n.alpha, n.w, n.b, out.rows, width, ctx->stream))
      return host->fail("%s", g_err);
    host->launched(ctx);
    return 0;
  }
};

extern "C" EngPart* make_dynamic_tanh(const EngHost* h, int width, const float* alpha, const float* w, const float* b) {
  host = h;
  return new DynamicTanh(width, TanhNorm{alpha, w, b});
}

extern "C" EngPart* make_normed_tokens(const EngHost* h, const void* table, int width, int dtype, float scale,
                                       const float* alpha, const float* w, const float* b) {
  host = h;
  NormedTokens* p = new NormedTokens;
  p->table = table, p->width = width, p->dtype = dtype, p->scale = scale, p->n = TanhNorm{alpha, w, b};
  return p;
}
