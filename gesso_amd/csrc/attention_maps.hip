// Attention as the difference of two softmax maps over one value row: the general kernel.
//
// Query head h has two queries of d features (columns [2 h d, (2 h + 2) d) of its row), its key head g = h / (nh / nkv) two
// keys a token, side by side in the key cache (num_pages, nkv, page_size, 2 d), and one value row a token in the value
// cache (num_pages, nkv, page_size, vd).  The query at position p sees the keys lo..p, lo = 0 or p - window + 1.
//
//   o_m = sum_u softmax_u((q_m . k_m,u) scale) v_u      for the maps m = 1, 2
//   o   = o_1 - lam o_2;   out = o / sqrt(mean(o^2) + eps) * out_scale * sigmoid(gate_h)
//
// The gate's logit stands in the query's row at column gate_col + h (gate_col < 0: no gate).  Any sizes up to 256 features
// a map and 512 a value, float32 or bfloat16 storage, float32 arithmetic.  One wavefront per (token, query head); keys in
// tiles of 64 from lo on with a running maximum and sum per map, so that a position's result does not depend on how its
// sequence was cut into steps.
#include "common.h"

#define AM_MAX_D 256
#define AM_MAX_VD 512

template <typename T>
__global__ void __launch_bounds__(64)
attention_maps_kernel(const T* __restrict__ q, int q_stride, const T* __restrict__ kcache, const T* __restrict__ vcache,
                      const int* __restrict__ positions, const int* __restrict__ seq_of_token,
                      const int* __restrict__ block_table, int max_blocks, int page_size, int window, float scale, float lam,
                      float eps, float out_scale, int gate_col, T* __restrict__ out, int nh, int nkv, int d, int vd) {
  __shared__ float qs[2 * AM_MAX_D];
  __shared__ float ps[2][64];
  __shared__ long rowoff[64];
  constexpr int NV = AM_MAX_VD / 64;
  const int lane = threadIdx.x, t = blockIdx.x, h = blockIdx.y;
  const int kvh = h / (nh / nkv);
  const int pos = positions[t];
  const int* bt = block_table + (size_t)seq_of_token[t] * max_blocks;
  const T* row = q + (size_t)t * q_stride;
  for (int j = lane; j < 2 * d; j += 64) qs[j] = to_f32(row[(size_t)h * 2 * d + j]);
  __syncthreads();
  const int lo = window > 0 && pos - window + 1 > 0 ? pos - window + 1 : 0;
  float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};
  float acc[2][NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) acc[0][i] = acc[1][i] = 0.f;

  for (int base = lo; base <= pos; base += 64) {
    const int u = base + lane;
    float s[2] = {-INFINITY, -INFINITY};
    long off = 0;
    if (u <= pos) {
      off = ((long)bt[u / page_size] * nkv + kvh) * page_size + u % page_size;
      const T* kr = kcache + off * 2 * d;
#pragma unroll
      for (int a = 0; a < 2; ++a) {
        float dot = 0.f;
        for (int j = 0; j < d; ++j) dot += qs[a * d + j] * to_f32(kr[a * d + j]);
        s[a] = dot * scale;
      }
    }
    float alpha[2], p[2];
#pragma unroll
    for (int a = 0; a < 2; ++a) {
      const float m_new = fmaxf(m[a], wave_max(s[a]));
      p[a] = u <= pos ? expf(s[a] - m_new) : 0.f;
      alpha[a] = expf(m[a] - m_new);       // 0 on the first tile (m = -inf), since m_new is finite there
      l[a] = l[a] * alpha[a] + wave_sum(p[a]);
      m[a] = m_new;
    }
    __syncthreads();
    ps[0][lane] = p[0];
    ps[1][lane] = p[1];
    rowoff[lane] = off;
    __syncthreads();
    const int nk = pos - base + 1 < 64 ? pos - base + 1 : 64;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int j = lane + 64 * i;
      if (j < vd) {
        float a0 = acc[0][i] * alpha[0], a1 = acc[1][i] * alpha[1];
        for (int k = 0; k < nk; ++k) {
          const float v = to_f32(vcache[rowoff[k] * vd + j]);
          a0 += ps[0][k] * v;
          a1 += ps[1][k] * v;
        }
        acc[0][i] = a0;
        acc[1][i] = a1;
      }
    }
  }
  const float inv0 = 1.f / l[0], inv1 = lam / l[1];
  float o[NV], ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    o[i] = lane + 64 * i < vd ? acc[0][i] * inv0 - acc[1][i] * inv1 : 0.f;
    ss += o[i] * o[i];
  }
  float f = norm_inverse(wave_sum(ss), (float)vd, eps) * out_scale;
  if (gate_col >= 0) f *= 1.f / (1.f + expf(-to_f32(row[gate_col + h])));
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int j = lane + 64 * i;
    if (j < vd) out[((size_t)t * nh + h) * vd + j] = from_f32<T>(o[i] * f);
  }
}

extern "C" int gs_attention_maps(const void* q, int q_stride, const void* kcache, const void* vcache, int dtype,
                                 const int* positions, const int* seq_of_token, const int* block_table, int max_blocks,
                                 int page_size, int window, float scale, float lam, float eps, float out_scale,
                                 int gate_col, void* out, int ntok, int nh, int nkv, int d, int vd, hipStream_t stream) {
  GS_REQUIRE(ntok >= 0 && nh > 0 && nkv > 0 && nh % nkv == 0, "attention_maps: bad sizes T=%d nh=%d nkv=%d", ntok, nh, nkv);
  GS_REQUIRE(d > 0 && d <= AM_MAX_D && vd > 0 && vd <= AM_MAX_VD, "attention_maps: maps of %d features and values of %d, the kernel holds up to %d and %d", d, vd, AM_MAX_D, AM_MAX_VD);
  GS_REQUIRE(nh <= 65535, "attention_maps: more than 65535 heads");
  GS_REQUIRE(page_size > 0 && max_blocks > 0 && window >= 0, "attention_maps: bad page_size/max_blocks/window");
  GS_REQUIRE(q_stride >= 2 * nh * d && (gate_col < 0 || gate_col + nh <= q_stride), "attention_maps: rows of %d hold no queries and gates", q_stride);
  GS_REQUIRE(eps > 0.f, "attention_maps: eps must be positive");
  if (ntok == 0) return 0;
  dim3 grid(ntok, nh);
#define GS_RUN(T)                                                                                                          \
  attention_maps_kernel<T><<<grid, 64, 0, stream>>>((const T*)q, q_stride, (const T*)kcache, (const T*)vcache, positions,  \
                                                    seq_of_token, block_table, max_blocks, page_size, window, scale, lam, \
                                                    eps, out_scale, gate_col, (T*)out, nh, nkv, d, vd)
  if (dtype == GS_F32)
    GS_RUN(float);
  else if (dtype == GS_BF16)
    GS_RUN(bf16);
  else
    GS_REQUIRE(false, "attention_maps: unknown dtype %d", dtype);
#undef GS_RUN
  GS_LAUNCH_CHECK("attention_maps");
  return 0;
}
