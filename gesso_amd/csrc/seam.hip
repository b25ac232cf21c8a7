// The seam between two sub-layers of a block that norms a sub-layer's output as well as its input, and the input a
// token brings to a layer of its own.
//
// norm_seam, one block per row r (source row s = rows ? rows[r] : r):
//   res[s] += mult * post(y[s])           (y may be absent: nothing is added)
//   out[r]  = pre(res[s])                 (out may be absent: nobody reads the row next)
// post and pre are each one of
//   0  the row as it is
//   1  rms:       x / sqrt(mean(x^2) + eps) * w
//   2  dyn_tanh:  tanh(alpha x) w + b, alpha one number on the device; no statistics of the row
// float32 arithmetic throughout.  A thread owns the same columns in every pass over the row, so what it wrote it may read
// again.  With `rows` (a gather at the model's end) nothing is added and res is left as it is.
//
// side_gate: out[t, j] = gelu_tanh(z[t, j]) * table[ids[t], offset + j] for j < dim, zeros in the spare columns behind.
#include "common.h"

#define SEAM_RAW 0
#define SEAM_RMS 1
#define SEAM_DYT 2

template <int V, typename T>
__device__ __forceinline__ void seam_load(const T* p, float* v) {
  if constexpr (V == 8) load8f(p, v);
  else v[0] = to_f32(p[0]);
}
template <int V, typename T>
__device__ __forceinline__ void seam_store(T* p, const float* v) {
  if constexpr (V == 8) store8f(p, v);
  else p[0] = from_f32<T>(v[0]);
}

template <typename TY, typename TO, int V>
__global__ void norm_seam_kernel(float* __restrict__ res, const TY* __restrict__ y, int post, const float* __restrict__ pw,
                                 const float* __restrict__ pb, const float* __restrict__ palpha, float peps, float mult,
                                 int pre, const float* __restrict__ qw, const float* __restrict__ qb,
                                 const float* __restrict__ qalpha, float qeps, TO* __restrict__ out,
                                 const int* __restrict__ rows, int H) {
  __shared__ float red[17];
  const int r = blockIdx.x, s = rows ? rows[r] : r;
  const int step = blockDim.x * V, j0 = threadIdx.x * V;
  float* x = res + (size_t)s * H;
  const TY* yr = y ? y + (size_t)s * H : nullptr;
  TO* o = out ? out + (size_t)r * H : nullptr;
  float pinv = 1.f;
  if (y && post == SEAM_RMS) {
    float ss = 0.f;
    for (int j = j0; j < H; j += step) {
      float v[V];
      seam_load<V>(yr + j, v);
#pragma unroll
      for (int e = 0; e < V; ++e) ss += v[e] * v[e];
    }
    pinv = norm_inverse(block_sum(ss, red), (float)H, peps);
  }
  const float pa = y && post == SEAM_DYT ? palpha[0] : 0.f, qa = o && pre == SEAM_DYT ? qalpha[0] : 0.f;
  float ss = 0.f;
  for (int j = j0; j < H; j += step) {
    float v[V], a[V], w[V], b[V];
    seam_load<V>(x + j, v);
    if (y) {
      seam_load<V>(yr + j, a);
      if (post != SEAM_RAW) seam_load<V>(pw + j, w);
      if (post == SEAM_DYT) {
        seam_load<V>(pb + j, b);
#pragma unroll
        for (int e = 0; e < V; ++e) a[e] = tanhf(pa * a[e]) * w[e] + b[e];
      } else if (post == SEAM_RMS) {
#pragma unroll
        for (int e = 0; e < V; ++e) a[e] = a[e] * pinv * w[e];
      }
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] += mult * a[e];
      seam_store<V>(x + j, v);
    }
    if (!o) continue;
    if (pre == SEAM_RMS) {
#pragma unroll
      for (int e = 0; e < V; ++e) ss += v[e] * v[e];
      continue;
    }
    if (pre == SEAM_DYT) {
      seam_load<V>(qw + j, w);
      seam_load<V>(qb + j, b);
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] = tanhf(qa * v[e]) * w[e] + b[e];
    }
    seam_store<V>(o + j, v);
  }
  if (!o || pre != SEAM_RMS) return;
  const float qinv = norm_inverse(block_sum(ss, red), (float)H, qeps);
  for (int j = j0; j < H; j += step) {
    float v[V], w[V];
    seam_load<V>(x + j, v);
    seam_load<V>(qw + j, w);
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] = v[e] * qinv * w[e];
    seam_store<V>(o + j, v);
  }
}

extern "C" int gs_norm_seam(float* res, const void* y, int y_dtype, int post, const float* pw, const float* pb,
                            const float* palpha, float peps, float mult, int pre, const float* qw, const float* qb,
                            const float* qalpha, float qeps, void* out, int out_dtype, const int* rows, int n_out, int H,
                            hipStream_t stream) {
  GS_REQUIRE(n_out >= 0 && H > 0, "norm_seam: bad sizes rows=%d H=%d", n_out, H);
  GS_REQUIRE(post >= SEAM_RAW && post <= SEAM_DYT && pre >= SEAM_RAW && pre <= SEAM_DYT, "norm_seam: unknown norms %d, %d", post, pre);
  GS_REQUIRE(!y || post == SEAM_RAW || (pw && (post == SEAM_RMS ? peps > 0.f : pb && palpha)), "norm_seam: the first norm lacks a tensor or its eps");
  GS_REQUIRE(!out || pre == SEAM_RAW || (qw && (pre == SEAM_RMS ? qeps > 0.f : qb && qalpha)), "norm_seam: the second norm lacks a tensor or its eps");
  GS_REQUIRE(!(rows && y), "norm_seam: chosen rows are read, not written");
  GS_REQUIRE(y || out, "norm_seam: nothing to do");
  if (n_out == 0) return 0;
  uintptr_t at = (uintptr_t)res | (uintptr_t)y | (uintptr_t)out;
  if (y && post != SEAM_RAW) at |= (uintptr_t)pw | (uintptr_t)pb;
  if (out && pre != SEAM_RAW) at |= (uintptr_t)qw | (uintptr_t)qb;
  const bool v8 = H % 8 == 0 && (at & 15) == 0;
  const int per = v8 ? 8 : 1, want = gs_ceil_div(gs_ceil_div(H, per), 64) * 64;
  const int threads = want < 64 ? 64 : (want > 512 ? 512 : want);
#define GS_RUN(TY, TO, V)                                                                                              \
  norm_seam_kernel<TY, TO, V><<<n_out, threads, 0, stream>>>(res, (const TY*)y, post, pw, pb, palpha, peps, mult, pre, \
                                                             qw, qb, qalpha, qeps, (TO*)out, rows, H)
#define GS_RUN_V(TY, TO)           \
  do {                             \
    if (v8) GS_RUN(TY, TO, 8);     \
    else GS_RUN(TY, TO, 1);        \
  } while (0)
  if (y_dtype == GS_F32 && out_dtype == GS_F32)
    GS_RUN_V(float, float);
  else if (y_dtype == GS_BF16 && out_dtype == GS_BF16)
    GS_RUN_V(bf16, bf16);
  else if (y_dtype == GS_F32 && out_dtype == GS_BF16)
    GS_RUN_V(float, bf16);
  else if (y_dtype == GS_BF16 && out_dtype == GS_F32)
    GS_RUN_V(bf16, float);
  else
    GS_REQUIRE(false, "norm_seam: unknown dtypes %d %d", y_dtype, out_dtype);
#undef GS_RUN_V
#undef GS_RUN
  GS_LAUNCH_CHECK("norm_seam");
  return 0;
}

template <typename TZ, typename TE, typename TO>
__global__ void side_gate_kernel(const TZ* __restrict__ z, int ldz, const TE* __restrict__ table, int ldt, int offset,
                                 const int* __restrict__ ids, int dim, TO* __restrict__ out, int width, long total) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= total) return;
  const long t = i / width;
  const int j = (int)(i - t * width);
  float v = 0.f;
  if (j < dim) {
    const float g = to_f32(z[t * ldz + j]), u = 0.7978845608028654f * (g + 0.044715f * g * g * g);
    v = 0.5f * g * (1.0f + tanhf(u)) * to_f32(table[(size_t)ids[t] * ldt + offset + j]);
  }
  out[i] = from_f32<TO>(v);
}

extern "C" int gs_side_gate(const void* z, int z_dtype, int ldz, const void* table, int table_dtype, int ldt, int offset,
                            const int* ids, int dim, void* out, int out_dtype, int width, int T, hipStream_t stream) {
  GS_REQUIRE(T >= 0 && dim > 0 && width >= dim && ldz >= dim, "side_gate: bad sizes T=%d dim=%d width=%d ldz=%d", T, dim, width, ldz);
  GS_REQUIRE(offset >= 0 && offset + dim <= ldt, "side_gate: columns %d + %d outside the table's rows of %d", offset, dim, ldt);
  if (T == 0) return 0;
  const long total = (long)T * width;
  const int blocks = gs_ceil_div(total, 256);
#define GS_RUN(TZ, TE, TO) \
  side_gate_kernel<TZ, TE, TO><<<blocks, 256, 0, stream>>>((const TZ*)z, ldz, (const TE*)table, ldt, offset, ids, dim, (TO*)out, width, total)
  if (z_dtype == GS_F32 && table_dtype == GS_F32 && out_dtype == GS_F32) GS_RUN(float, float, float);
  else if (z_dtype == GS_F32 && table_dtype == GS_BF16 && out_dtype == GS_BF16) GS_RUN(float, bf16, bf16);
  else if (z_dtype == GS_F32 && table_dtype == GS_F32 && out_dtype == GS_BF16) GS_RUN(float, float, bf16);
  else if (z_dtype == GS_BF16 && table_dtype == GS_BF16 && out_dtype == GS_BF16) GS_RUN(bf16, bf16, bf16);
  else if (z_dtype == GS_BF16 && table_dtype == GS_F32 && out_dtype == GS_BF16) GS_RUN(bf16, float, bf16);
  else GS_REQUIRE(false, "side_gate: unknown dtypes %d %d %d", z_dtype, table_dtype, out_dtype);
#undef GS_RUN
  GS_LAUNCH_CHECK("side_gate");
  return 0;
}
