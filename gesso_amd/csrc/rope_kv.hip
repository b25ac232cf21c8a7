// Per-head RMSNorm of q and k, rotary position encoding, and the write of K and V into the cache pages.
//
// qkv (T, (nh + 2 nkv) d): q heads, then k heads, then v heads, each head d wide.
//   q, k: x = x / sqrt(mean(x^2) + eps) * w  over the head (when a weight is given), then for the
//         first rotary_dim features, pairs (a, b) = (i, i + rotary_dim/2) ("half-split") or, with `interleaved`,
//         (2i, 2i + 1) (reference src/Operators/cpu.jl:357-371):
//           x_a' = x_a cos - x_b sin,  x_b' = x_a sin + x_b cos,  angle = pos * theta^(-2i/rotary_dim)
//         with cos/sin row i from a table (max_position, rotary_dim/2) made on the host in float64.
//   q is written back in place; k (after norm and rotation) and v (as it is) go to the cache:
//   page = block_table[seq, pos / page_size], row = pos % page_size,
//   cache (num_pages, nkv, page_size, d).
// A value head may be vd wide instead of d (the row is then (nh + nkv) d + nkv vd wide, the value cache
// (num_pages, nkv, page_size, vd)), and with value tables (max_position, vd/2) the values are cached turned by
// their own position over their whole width, in the same layout of pairs; whoever sums them turns the sum back.
// The rows may be wider than q|k|v (`ld` values apart: further products of the same input stand behind them).
// `plain_norm`: q and k are divided by their root mean square without a weight (a turn keeps a head's sum of squares,
// so the same numbers come out whether the division stands before or after it).  `v_first` (rows `ldf` apart, the value
// heads from column 0 on) with `mix` (one float on the device): the values are cached as (1 - mix) v + mix v_first.
// `maps` > 1: a value head goes with that many keys of width d (the rows hold nkv maps key heads before the nkv value heads,
// key head by key head, its maps side by side); the key cache is (num_pages, nkv, page_size, maps d), a head's keys of a
// token side by side.
// One wave per (token, head).  All arithmetic float32.
#include "common.h"

template <typename T>
__global__ void qknorm_rope_kv_kernel(T* __restrict__ qkv, const float* __restrict__ qw, const float* __restrict__ kw,
                                      float eps, const float* __restrict__ cos_t, const float* __restrict__ sin_t,
                                      int rotary_dim, int interleaved, const int* __restrict__ positions,
                                      const int* __restrict__ seq_of_token, const int* __restrict__ block_table,
                                      int max_blocks, int page_size, T* __restrict__ kcache, T* __restrict__ vcache,
                                      int ntok, int nh, int nkv, int d, int write_kv, int vd,
                                      const float* __restrict__ vcos, const float* __restrict__ vsin, int ld,
                                      int plain_norm, const T* __restrict__ v_first, int ldf,
                                      const float* __restrict__ mix, int maps) {
  int lane = threadIdx.x & 63;
  const int nk = nkv * maps;
  int heads = nh + nk + nkv;
  long unit = (long)blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (unit >= (long)ntok * heads) return;
  int t = (int)(unit / heads);
  int hh = (int)(unit - (long)t * heads);
  const size_t row_len = (size_t)ld;
  const bool is_v = hh >= nh + nk;
  T* x = qkv + (size_t)t * row_len + (is_v ? (size_t)(nh + nk) * d + (size_t)(hh - nh - nk) * vd : (size_t)hh * d);
  int pos = positions[t];

  T* dst = nullptr;  // cache row for k and v heads
  if (hh >= nh) {
    if (!write_kv) return;
    int kvh = is_v ? hh - nh - nk : hh - nh, map = 0;
    if (!is_v && maps > 1) {
      map = kvh % maps;
      kvh /= maps;
    }
    int page = block_table[(size_t)seq_of_token[t] * max_blocks + pos / page_size];
    T* base = is_v ? vcache : kcache;
    dst = base + (((size_t)page * nkv + kvh) * page_size + pos % page_size) * (is_v ? vd : maps * d) + map * d;
  }
  if (is_v) {  // v: copy, blend with another layer's values, or turn by the position over the whole width
    if (v_first) {
      const float lam = mix[0];
      const T* f = v_first + (size_t)t * ldf + (size_t)(hh - nh - nk) * vd;
      for (int j = lane; j < vd; j += 64) dst[j] = from_f32<T>((1.f - lam) * to_f32(x[j]) + lam * to_f32(f[j]));
      return;
    }
    if (!vcos) {
      for (int j = lane; j < vd; j += 64) dst[j] = x[j];
      return;
    }
    const int vh = vd >> 1;
    for (int i = lane; i < vh; i += 64) {
      const int ia = interleaved ? 2 * i : i, ib = interleaved ? 2 * i + 1 : i + vh;
      const float a = to_f32(x[ia]), b = to_f32(x[ib]);
      const float c = vcos[(size_t)pos * vh + i], s = vsin[(size_t)pos * vh + i];
      dst[ia] = from_f32<T>(a * c - b * s);
      dst[ib] = from_f32<T>(a * s + b * c);
    }
    return;
  }

  const float* w = hh < nh ? qw : kw;
  float inv = 1.f;
  if (w || plain_norm) {
    float ss = 0.f;
    for (int j = lane; j < d; j += 64) {
      float v = to_f32(x[j]);
      ss += v * v;
    }
    ss = wave_sum(ss);
    inv = norm_inverse(ss, (float)d, eps);
  }
  T* o = hh < nh ? x : dst;
  int half = rotary_dim >> 1;
  const float* cr = cos_t ? cos_t + (size_t)pos * half : nullptr;
  const float* sr = sin_t ? sin_t + (size_t)pos * half : nullptr;
  for (int i = lane; i < half; i += 64) {
    const int ia = interleaved ? 2 * i : i, ib = interleaved ? 2 * i + 1 : i + half;
    float a = to_f32(x[ia]) * inv, b = to_f32(x[ib]) * inv;
    if (w) {
      a *= w[ia];
      b *= w[ib];
    }
    float c = cr[i], s = sr[i];
    o[ia] = from_f32<T>(a * c - b * s);
    o[ib] = from_f32<T>(a * s + b * c);
  }
  for (int j = rotary_dim + lane; j < d; j += 64) {  // features beyond the rotary part
    float a = to_f32(x[j]) * inv;
    if (w) a *= w[j];
    o[j] = from_f32<T>(a);
  }
}

// The same for head widths of 16, 32, 64 and 128 that are rotated whole (rotary_dim == d): L = d / 8 lanes per
// (token, head), eight features a lane, 16-byte loads and stores; the halves of a rotation pair sit L/2 lanes apart.
template <typename T, int L>
__global__ void qknorm_rope_kv_vec_kernel(T* __restrict__ qkv, const float* __restrict__ qw,
                                          const float* __restrict__ kw, float eps, const float* __restrict__ cos_t,
                                          const float* __restrict__ sin_t, const int* __restrict__ positions,
                                          const int* __restrict__ seq_of_token, const int* __restrict__ block_table,
                                          int max_blocks, int page_size, T* __restrict__ kcache,
                                          T* __restrict__ vcache, int ntok, int nh, int nkv, int write_kv) {
  constexpr int d = 8 * L, half = d / 2;
  const int heads = nh + 2 * nkv;
  const long unit = ((long)blockIdx.x * blockDim.x + threadIdx.x) / L;
  const int sub = threadIdx.x % L;
  const bool live = unit < (long)ntok * heads;   // lanes past the end run along for the shuffles, on unit 0
  const long un = live ? unit : 0;
  const int t = (int)(un / heads);
  const int hh = (int)(un - (long)t * heads);
  T* x = qkv + ((size_t)t * heads + hh) * d + sub * 8;
  const int pos = positions[t];
  const bool is_q = hh < nh, is_k = !is_q && hh < nh + nkv;
  T* o = x;
  if (!is_q) {
    const int kvh = is_k ? hh - nh : hh - nh - nkv;
    const int page = block_table[(size_t)seq_of_token[t] * max_blocks + pos / page_size];
    o = (is_k ? kcache : vcache) + (((size_t)page * nkv + kvh) * page_size + pos % page_size) * d + sub * 8;
  }
  float v[8];
  load8f(x, v);
  if (is_q || is_k) {
    const float* w = is_q ? qw : kw;
    if (w) {
      float ss = 0.f;
#pragma unroll
      for (int k = 0; k < 8; ++k) ss += v[k] * v[k];
#pragma unroll
      for (int m = 1; m < L; m <<= 1) ss += __shfl_xor(ss, m, 64);
      const float inv = norm_inverse(ss, (float)d, eps);
      float w8[8];
      load8f(w + sub * 8, w8);
#pragma unroll
      for (int k = 0; k < 8; ++k) v[k] = v[k] * inv * w8[k];
    }
    const bool low = sub < L / 2;                 // holds the first halves (i) of its pairs, else the second (j)
    const int i0 = (low ? sub : sub - L / 2) * 8;
    float c8[8], s8[8];
    load8f(cos_t + (size_t)pos * half + i0, c8);
    load8f(sin_t + (size_t)pos * half + i0, s8);
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      const float other = __shfl_xor(v[k], L / 2, 64);
      // x_i' = x_i cos - x_j sin,  x_j' = x_i sin + x_j cos
      v[k] = low ? v[k] * c8[k] - other * s8[k] : other * s8[k] + v[k] * c8[k];
    }
  }
  if (live && (is_q || write_kv)) store8f(o, v);
}

// Heads of other widths in whole pieces of eight, or rotated in part (rotary_dim a multiple of 16, half-split): P lanes per
// (token, head), a power of two, of which the first d / 8 hold eight features each; a feature's partner lies rotary_dim / 16
// lanes away, and lanes beyond the rotary part keep theirs.
template <typename T, int P>
__global__ void qknorm_rope_kv_part_kernel(T* __restrict__ qkv, const float* __restrict__ qw, const float* __restrict__ kw,
                                           float eps, const float* __restrict__ cos_t, const float* __restrict__ sin_t,
                                           int rotary_dim, const int* __restrict__ positions,
                                           const int* __restrict__ seq_of_token, const int* __restrict__ block_table,
                                           int max_blocks, int page_size, T* __restrict__ kcache, T* __restrict__ vcache,
                                           int ntok, int nh, int nkv, int d, int write_kv, int ld) {
  const int heads = nh + 2 * nkv;
  const long unit = ((long)blockIdx.x * blockDim.x + threadIdx.x) / P;
  const int sub = threadIdx.x % P;
  const bool live = unit < (long)ntok * heads && sub * 8 < d;   // the others run along for the shuffles
  const long un = unit < (long)ntok * heads ? unit : 0;
  const int t = (int)(un / heads);
  const int hh = (int)(un - (long)t * heads);
  T* x = qkv + (size_t)t * ld + (size_t)hh * d + sub * 8;
  const int pos = positions[t];
  const bool is_q = hh < nh, is_k = !is_q && hh < nh + nkv;
  T* o = x;
  if (!is_q) {
    const int kvh = is_k ? hh - nh : hh - nh - nkv;
    const int page = block_table[(size_t)seq_of_token[t] * max_blocks + pos / page_size];
    o = (is_k ? kcache : vcache) + (((size_t)page * nkv + kvh) * page_size + pos % page_size) * d + sub * 8;
  }
  float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
  if (live) load8f(x, v);
  if (qw) {
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < 8; ++k) ss += v[k] * v[k];
#pragma unroll
    for (int m = 1; m < P; m <<= 1) ss += __shfl_xor(ss, m, 64);
    if (live && (is_q || is_k)) {
      const float inv = norm_inverse(ss, (float)d, eps);
      float w8[8];
      load8f((is_q ? qw : kw) + sub * 8, w8);
#pragma unroll
      for (int k = 0; k < 8; ++k) v[k] = v[k] * inv * w8[k];
    }
  }
  const int hp = rotary_dim >> 4, half = rotary_dim >> 1;       // lanes a half of the rotary part takes
  const bool low = sub < hp, turned = sub < 2 * hp;
  const int from = (threadIdx.x & 63) + (turned ? (low ? hp : -hp) : 0);
  float other[8];
#pragma unroll
  for (int k = 0; k < 8; ++k) other[k] = __shfl(v[k], from, 64);
  if (!live || (!is_q && !write_kv)) return;
  if (turned && (is_q || is_k)) {
    float c8[8], s8[8];
    const int i0 = (low ? sub : sub - hp) * 8;
    load8f(cos_t + (size_t)pos * half + i0, c8);
    load8f(sin_t + (size_t)pos * half + i0, s8);
#pragma unroll
    for (int k = 0; k < 8; ++k) v[k] = low ? v[k] * c8[k] - other[k] * s8[k] : other[k] * s8[k] + v[k] * c8[k];
  }
  store8f(o, v);
}

extern "C" int gs_qknorm_rope_kv(void* qkv, int dtype, const float* qw, const float* kw, float eps,
                                 const float* cos_t, const float* sin_t, int rotary_dim, int interleaved,
                                 int max_position, const int* positions, const int* seq_of_token, const int* block_table,
                                 int max_blocks, int page_size, void* kcache, void* vcache, int ntok, int nh, int nkv,
                                 int d, int write_kv, int vd, const float* vcos, const float* vsin, int ld,
                                 int plain_norm, const void* v_first, int ldf, const float* mix, int maps,
                                 hipStream_t stream) {
  GS_REQUIRE(maps >= 1 && maps <= 64, "qknorm_rope_kv: %d keys a head", maps);
  GS_REQUIRE(vd > 0, "qknorm_rope_kv: values of width %d", vd);
  GS_REQUIRE((vcos == nullptr) == (vsin == nullptr), "qknorm_rope_kv: the value tables come together");
  GS_REQUIRE(!vcos || (vd % 2 == 0 && max_position > 0), "qknorm_rope_kv: turned values are of even width");
  GS_REQUIRE(ntok >= 0 && nh > 0 && nkv > 0 && d > 0, "qknorm_rope_kv: bad sizes T=%d nh=%d nkv=%d d=%d", ntok, nh,
             nkv, d);
  GS_REQUIRE(rotary_dim >= 0 && rotary_dim <= d && rotary_dim % 2 == 0,
             "qknorm_rope_kv: rotary_dim %d must be even and at most the head width %d", rotary_dim, d);
  GS_REQUIRE(rotary_dim == 0 || (cos_t && sin_t && max_position > 0), "qknorm_rope_kv: rotation without a table");
  GS_REQUIRE(page_size > 0 && max_blocks > 0, "qknorm_rope_kv: bad page_size %d or max_blocks %d", page_size,
             max_blocks);
  GS_REQUIRE((qw == nullptr) == (kw == nullptr), "qknorm_rope_kv: q and k norm weights come together");
  const int narrow = (nh + nkv * maps) * d + nkv * vd;
  if (ld == 0) ld = narrow;
  GS_REQUIRE(ld >= narrow, "qknorm_rope_kv: rows of %d values do not hold q, k and v (%d)", ld, narrow);
  GS_REQUIRE(!(plain_norm && qw), "qknorm_rope_kv: a head norm has a weight or none");
  GS_REQUIRE((v_first == nullptr) == (mix == nullptr) && (!v_first || (ldf >= nkv * vd && !vcos)),
             "qknorm_rope_kv: blended values need the other values (rows of at least %d) and the share", nkv * vd);
  if (ntok == 0) return 0;
  long units = (long)ntok * (nh + nkv * maps + nkv);
  const bool vec = maps == 1 && ld == narrow && !plain_norm && !v_first && !interleaved && vd == d && !vcos && rotary_dim == d && (d == 16 || d == 32 || d == 64 || d == 128) && (dtype == GS_F32 || dtype == GS_BF16) &&
                   ((uintptr_t)qkv & 15) == 0 && ((uintptr_t)kcache & 15) == 0 && ((uintptr_t)vcache & 15) == 0 &&
                   ((uintptr_t)cos_t & 15) == 0 && ((uintptr_t)sin_t & 15) == 0 && ((uintptr_t)qw & 15) == 0 &&
                   ((uintptr_t)kw & 15) == 0;
  if (vec) {
    const int L = d / 8;
    const int vblocks = gs_ceil_div(units * L, 256);
#define GS_VEC(T, LL)                                                                                              \
  qknorm_rope_kv_vec_kernel<T, LL><<<vblocks, 256, 0, stream>>>((T*)qkv, qw, kw, eps, cos_t, sin_t, positions,     \
                                                                seq_of_token, block_table, max_blocks, page_size, \
                                                                (T*)kcache, (T*)vcache, ntok, nh, nkv, write_kv)
#define GS_VEC_T(T)                                                                     \
  switch (L) {                                                                          \
    case 2: GS_VEC(T, 2); break;                                                        \
    case 4: GS_VEC(T, 4); break;                                                        \
    case 8: GS_VEC(T, 8); break;                                                        \
    default: GS_VEC(T, 16); break;                                                      \
  }
    if (dtype == GS_F32) { GS_VEC_T(float) } else { GS_VEC_T(bf16) }
#undef GS_VEC_T
#undef GS_VEC
    GS_LAUNCH_CHECK("qknorm_rope_kv");
    return 0;
  }
  const bool part = maps == 1 && !plain_norm && !v_first && !interleaved && vd == d && !vcos && d % 8 == 0 && d <= 256 &&
                    rotary_dim % 16 == 0 && ld % 8 == 0 && (dtype == GS_F32 || dtype == GS_BF16) &&
                    (((uintptr_t)qkv | (uintptr_t)kcache | (uintptr_t)vcache | (uintptr_t)cos_t | (uintptr_t)sin_t |
                      (uintptr_t)qw | (uintptr_t)kw) & 15) == 0;
  if (part) {
    int P = 1;
    while (P * 8 < d) P *= 2;
    const int pblocks = gs_ceil_div(units * P, 256);
#define GS_PART(T, PP)                                                                                                     \
  qknorm_rope_kv_part_kernel<T, PP><<<pblocks, 256, 0, stream>>>((T*)qkv, qw, kw, eps, cos_t, sin_t, rotary_dim, positions, \
                                                                 seq_of_token, block_table, max_blocks, page_size,         \
                                                                 (T*)kcache, (T*)vcache, ntok, nh, nkv, d, write_kv, ld)
#define GS_PART_T(T)                   \
  switch (P) {                         \
    case 1: GS_PART(T, 1); break;      \
    case 2: GS_PART(T, 2); break;      \
    case 4: GS_PART(T, 4); break;      \
    case 8: GS_PART(T, 8); break;      \
    case 16: GS_PART(T, 16); break;    \
    default: GS_PART(T, 32); break;    \
  }
    if (dtype == GS_F32) { GS_PART_T(float) } else { GS_PART_T(bf16) }
#undef GS_PART_T
#undef GS_PART
    GS_LAUNCH_CHECK("qknorm_rope_kv");
    return 0;
  }
  int blocks = gs_ceil_div(units, 4);
#define GS_RUN(T)                                                                                               \
  qknorm_rope_kv_kernel<T><<<blocks, 256, 0, stream>>>((T*)qkv, qw, kw, eps, cos_t, sin_t, rotary_dim, interleaved, positions, \
                                                       seq_of_token, block_table, max_blocks, page_size,        \
                                                       (T*)kcache, (T*)vcache, ntok, nh, nkv, d, write_kv, vd, vcos, vsin, \
                                                       ld, plain_norm, (const T*)v_first, ldf, mix, maps)
  if (dtype == GS_F32)
    GS_RUN(float);
  else if (dtype == GS_BF16)
    GS_RUN(bf16);
  else
    GS_REQUIRE(false, "qknorm_rope_kv: unknown dtype %d", dtype);
#undef GS_RUN
  GS_LAUNCH_CHECK("qknorm_rope_kv");
  return 0;
}

// Rows of heads turned in place by their tokens' positions, backwards with sign < 0: x (T, nh, w), every head over its
// whole width, pairs (i, i + w/2) or, with `interleaved`, (2i, 2i + 1); tables (max_position, w/2).  What attention
// over values that were cached turned needs at its end: each head's sum turned back by the query's position.
template <typename T>
__global__ void turn_heads_kernel(T* __restrict__ x, const float* __restrict__ cos_t, const float* __restrict__ sin_t,
                                  const int* __restrict__ positions, int interleaved, float sign, long units, int nh, int w) {
  const int lane = threadIdx.x & 63;
  const long unit = (long)blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (unit >= units) return;
  const int t = (int)(unit / nh);
  T* row = x + (size_t)unit * w;
  const int half = w >> 1;
  const float* cr = cos_t + (size_t)positions[t] * half;
  const float* sr = sin_t + (size_t)positions[t] * half;
  for (int i = lane; i < half; i += 64) {
    const int ia = interleaved ? 2 * i : i, ib = interleaved ? 2 * i + 1 : i + half;
    const float a = to_f32(row[ia]), b = to_f32(row[ib]);
    const float c = cr[i], s = sign * sr[i];
    row[ia] = from_f32<T>(a * c - b * s);
    row[ib] = from_f32<T>(a * s + b * c);
  }
}

extern "C" int gs_turn_heads(void* x, int dtype, const float* cos_t, const float* sin_t, int max_position,
                             const int* positions, int interleaved, float sign, int ntok, int nh, int w,
                             hipStream_t stream) {
  GS_REQUIRE(ntok >= 0 && nh > 0 && w > 0 && w % 2 == 0, "turn_heads: bad sizes T=%d nh=%d w=%d", ntok, nh, w);
  GS_REQUIRE(cos_t && sin_t && max_position > 0, "turn_heads: no tables");
  if (ntok == 0) return 0;
  const long units = (long)ntok * nh;
  const int blocks = gs_ceil_div(units, 4);
  if (dtype == GS_F32)
    turn_heads_kernel<float><<<blocks, 256, 0, stream>>>((float*)x, cos_t, sin_t, positions, interleaved, sign, units, nh, w);
  else if (dtype == GS_BF16)
    turn_heads_kernel<bf16><<<blocks, 256, 0, stream>>>((bf16*)x, cos_t, sin_t, positions, interleaved, sign, units, nh, w);
  else
    GS_REQUIRE(false, "turn_heads: unknown dtype %d", dtype);
  GS_LAUNCH_CHECK("turn_heads");
  return 0;
}
