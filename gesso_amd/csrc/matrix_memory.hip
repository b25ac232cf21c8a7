// What a matrix memory with exponential gates computes around its recurrence (gated_recurrence.hip walks the memory itself).
//
// exp_gates: per token and head, from the products z (T, ldz) float32 (the input gate's at [oi + h], the forget gate's at
// [of + h]), biases added,
//   i = cap tanh(zi / cap),   f = log sigmoid(cap tanh(zf / cap))
//   p_t = max(f_t + p_(t-1), i_t)                        a running maximum, the request's own, kept in its slot
//   gates[t, h] = exp(f + p_(t-1) - p_t)                 what the memory keeps
//   gates[t, H + h] = exp(i - p_t)                       with what the token is written
//   gates[t, 2 H + h] = exp(-p_t)                        the least the output is divided by
// With `logs` the first two are their base-2 logarithms instead.  A token takes the maximum from p to max(p + f, i), and such
// maps compose, (f1, i1) then (f2, i2) = (f1 + f2, max(i1 + f2, i2)), so six steps between lanes give 64 tokens' p.  Steps of
// few tokens: a wavefront per (sequence, head), four heads a block.  Longer portions: a block per (sequence, head), whose
// wavefronts take 64 tokens each and hand their maps on through LDS.
//
// memory_step: one token a sequence.  A step then reads and writes every state once, and that stream is all the work: a block
// owns 64 value columns of a (sequence, head), a wavefront a quarter of the rows, a lane a column, so that a row's columns
// are read and written side by side; the wavefronts' shares of S^T q are added in order.  The state's last column (the sum of
// the keys) goes along in the first column block, a thread a row.
//
// memory_outnorm: a head's m columns o and the number n . q (`den`), float32:
//   u = o / (max(|n . q|, exp(-p)) + 1e-6);   out = u / sqrt(mean(u^2) + eps) * w * sigmoid(gate)      per head
// Head h of token t has its columns at o[(t H + h) hs] and its number at den[(t H + h) ds].
#include "common.h"

#define MM_LOG2E 1.4426950408889634f

// W wavefronts share a (sequence, head); W = 1: each of the block's four has a head of its own.
template <int W>
__global__ void __launch_bounds__(W == 1 ? 256 : W * 64)
exp_gates_kernel(const float* __restrict__ z, int ldz, int oi, int of, const float* __restrict__ bi,
                 const float* __restrict__ bf, float cap, float* __restrict__ peak, const int* __restrict__ q_start,
                 const int* __restrict__ slots, float* __restrict__ gates, int H, int logs) {
  __shared__ float wf[W], wi[W];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, seq = blockIdx.x;
  const int h = W == 1 ? blockIdx.y * 4 + wave : blockIdx.y;
  if (h >= H) return;                                // (with W > 1 there is a block per head: all of it or nothing)
  const int t0 = q_start[seq], t1 = q_start[seq + 1];
  if (t1 <= t0) return;
  float* own = peak + (size_t)slots[seq] * H + h;
  float p = *own;
  const float b_i = bi[h], b_f = bf[h], inv_cap = 1.0f / cap;
  for (int tb = t0; tb < t1; tb += 64 * W) {
    const int t = tb + (W == 1 ? lane : (int)threadIdx.x);
    const bool in = t < t1;
    float f = 0.f, i = -INFINITY;                    // (a lane without a token: the map that changes nothing)
    if (in) {
      const float zi = z[(size_t)t * ldz + oi + h] + b_i, zf = z[(size_t)t * ldz + of + h] + b_f;
      i = cap * tanhf(zi * inv_cap);
      const float u = cap * tanhf(zf * inv_cap);
      f = fminf(u, 0.f) - log1pf(expf(-fabsf(u)));
    }
    float F = f, M = i;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float Fb = __shfl_up(F, o, 64), Mb = __shfl_up(M, o, 64);
      if (lane >= o) {
        M = fmaxf(Mb + F, M);
        F += Fb;
      }
    }
    float start = p;                                 // the maximum before this wavefront's tokens
    if constexpr (W > 1) {
      __syncthreads();                               // (the turn before has been read)
      if (lane == 63) {
        wf[wave] = F;
        wi[wave] = M;
      }
      __syncthreads();
#pragma unroll
      for (int w = 0; w < W; ++w) {
        if (w == wave) start = p;
        p = fmaxf(p + wf[w], wi[w]);
      }
    } else {
      p = fmaxf(p + __shfl(F, 63, 64), __shfl(M, 63, 64));
    }
    const float now = fmaxf(start + F, M);
    const float up = __shfl_up(now, 1, 64), before = lane == 0 ? start : up;
    if (in) {
      float* g = gates + (size_t)t * 3 * H + h;
      const float keep = f + before - now, put = i - now;
      g[0] = logs ? keep * MM_LOG2E : expf(keep);
      g[H] = logs ? put * MM_LOG2E : expf(put);
      g[2 * H] = expf(-now);
    }
  }
  if (W == 1 ? lane == 0 : threadIdx.x == 0) *own = p;
}

// longest: the most tokens a sequence brings (how a launch is shaped, not what it computes)
extern "C" int gs_exp_gates(const float* z, int ldz, int oi, int of, const float* bi, const float* bf, float cap, float* peak,
                            const int* q_start, const int* slots, float* gates, int nseq, int H, int longest, int logs,
                            hipStream_t stream) {
  GS_REQUIRE(nseq >= 0 && H > 0 && H <= 65535, "exp_gates: bad sizes nseq=%d H=%d", nseq, H);
  GS_REQUIRE(oi >= 0 && of >= 0 && oi + H <= ldz && of + H <= ldz, "exp_gates: the gates' products lie outside the rows of %d", ldz);
  GS_REQUIRE(cap > 0.f, "exp_gates: the cap must be positive");
  if (nseq == 0) return 0;
#define GS_RUN(W, BLOCKS)                                                                                                   \
  exp_gates_kernel<W><<<dim3(nseq, BLOCKS), W == 1 ? 256 : W * 64, 0, stream>>>(z, ldz, oi, of, bi, bf, cap, peak, q_start, \
                                                                                slots, gates, H, logs)
  if (longest <= 64) GS_RUN(1, gs_ceil_div(H, 4));
  else if (longest <= 512) GS_RUN(4, H);
  else GS_RUN(16, H);
#undef GS_RUN
  GS_LAUNCH_CHECK("exp_gates");
  return 0;
}

#define MS_U 16           // rows a lane has in flight
template <typename T>
__global__ void __launch_bounds__(256)
memory_step_kernel(const T* __restrict__ x, int ld, int oq, int ok, int ov, float q_scale, const float* __restrict__ gates,
                   float* __restrict__ state, const int* __restrict__ slots, float* __restrict__ out,
                   float* __restrict__ den, int H, int n, int m) {
  extern __shared__ float ms_qk[];                    // q, then the weighted key, n each
  __shared__ float part[4][64], red[17];
  const int seq = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int j = blockIdx.z * 64 + lane, ms = m + 1;
  const T* row = x + (size_t)seq * ld;
  const float* g = gates + (size_t)seq * 3 * H + h;
  const float keep = g[0], put = g[H];
  float* S = state + ((size_t)slots[seq] * H + h) * n * ms;
  float* q = ms_qk;
  float* k = ms_qk + n;
  for (int i = threadIdx.x; i < n; i += 256) {
    q[i] = to_f32(row[oq + h * n + i]) * q_scale;
    k[i] = to_f32(row[ok + h * n + i]) * put;
  }
  const bool col = j < m;
  const float v = col ? to_f32(row[ov + h * m + j]) : 0.f;
  __syncthreads();
  const int per = (n + 3) / 4, i0 = wave * per, i1 = i0 + per < n ? i0 + per : n;
  float acc = 0.f;
  if (col) {
    for (int ib = i0; ib < i1; ib += MS_U) {
      float s[MS_U];
#pragma unroll
      for (int u = 0; u < MS_U; ++u) s[u] = S[(size_t)(ib + u < i1 ? ib + u : ib) * ms + j];
#pragma unroll
      for (int u = 0; u < MS_U; ++u) {
        if (ib + u < i1) {
          const float w = fmaf(k[ib + u], v, keep * s[u]);
          S[(size_t)(ib + u) * ms + j] = w;
          acc = fmaf(w, q[ib + u], acc);
        }
      }
    }
  }
  part[wave][lane] = acc;
  float d = 0.f;
  if (blockIdx.z == 0)
    for (int i = threadIdx.x; i < n; i += 256) {
      const float w = fmaf(keep, S[(size_t)i * ms + m], k[i]);
      S[(size_t)i * ms + m] = w;
      d = fmaf(w, q[i], d);
    }
  __syncthreads();
  if (wave == 0 && col) out[((size_t)seq * H + h) * m + j] = (part[0][lane] + part[1][lane]) + (part[2][lane] + part[3][lane]);
  if (blockIdx.z == 0) {
    d = block_sum(d, red);
    if (threadIdx.x == 0) den[(size_t)seq * H + h] = d;
  }
}

extern "C" int gs_memory_step(const void* x, int dtype, int ld, int oq, int ok, int ov, float q_scale, const float* gates,
                              float* state, const int* slots, float* out, float* den, int nseq, int H, int n, int m,
                              hipStream_t stream) {
  GS_REQUIRE(nseq >= 0 && H > 0 && H <= 65535 && n > 0 && n <= 4096 && m > 0 && gs_ceil_div(m, 64) <= 65535,
             "memory_step: bad sizes nseq=%d H=%d n=%d m=%d", nseq, H, n, m);
  GS_REQUIRE(oq >= 0 && ok >= 0 && ov >= 0 && oq + H * n <= ld && ok + H * n <= ld && ov + H * m <= ld,
             "memory_step: q, k or v lie outside the rows of %d", ld);
  if (nseq == 0) return 0;
  dim3 grid(nseq, H, gs_ceil_div(m, 64));
  const size_t lds = 2 * (size_t)n * sizeof(float);
  if (dtype == GS_F32)
    memory_step_kernel<float><<<grid, 256, lds, stream>>>((const float*)x, ld, oq, ok, ov, q_scale, gates, state, slots, out, den, H, n, m);
  else if (dtype == GS_BF16)
    memory_step_kernel<bf16><<<grid, 256, lds, stream>>>((const bf16*)x, ld, oq, ok, ov, q_scale, gates, state, slots, out, den, H, n, m);
  else
    GS_REQUIRE(false, "memory_step: unknown dtype %d", dtype);
  GS_LAUNCH_CHECK("memory_step");
  return 0;
}

// One block per token, a wavefront per head in turn; a lane's columns are c = lane, lane + 64, ...: up to MM_KEEP of them
// stay in registers between the two passes.
#define MM_KEEP 8
template <typename TG, typename TO>
__global__ void __launch_bounds__(256)
memory_outnorm_kernel(const float* __restrict__ o, int hs, const float* __restrict__ den, int ds,
                      const float* __restrict__ gates, const TG* __restrict__ rows, int ldr,
                      int og, const float* __restrict__ w, float eps, TO* __restrict__ out, int H, int m) {
  const int t = blockIdx.x, lane = threadIdx.x & 63, nw = blockDim.x >> 6;
  for (int h = threadIdx.x >> 6; h < H; h += nw) {
    const float* row = o + ((size_t)t * H + h) * hs;
    const TG* gt = rows + (size_t)t * ldr + og + (size_t)h * m;
    const float inv_den = 1.0f / (fmaxf(fabsf(den[((size_t)t * H + h) * ds]), gates[(size_t)t * 3 * H + 2 * H + h]) + 1e-6f);
    float keep[MM_KEEP], ss = 0.f;
#pragma unroll
    for (int u = 0; u < MM_KEEP; ++u) {
      const int c = lane + 64 * u;
      keep[u] = c < m ? row[c] * inv_den : 0.f;
      ss += keep[u] * keep[u];
    }
    for (int c = lane + 64 * MM_KEEP; c < m; c += 64) {
      const float v = row[c] * inv_den;
      ss += v * v;
    }
    const float inv = norm_inverse(wave_sum(ss), (float)m, eps);
    TO* dst = out + ((size_t)t * H + h) * m;
    const float* wh = w + (size_t)h * m;
#pragma unroll
    for (int u = 0; u < MM_KEEP; ++u) {
      const int c = lane + 64 * u;
      if (c < m) dst[c] = from_f32<TO>(keep[u] * inv * wh[c] / (1.0f + expf(-to_f32(gt[c]))));
    }
    for (int c = lane + 64 * MM_KEEP; c < m; c += 64)
      dst[c] = from_f32<TO>(row[c] * inv_den * inv * wh[c] / (1.0f + expf(-to_f32(gt[c]))));
  }
}

extern "C" int gs_memory_outnorm(const float* o, int hs, const float* den, int ds, const float* gates, const void* rows, int rows_dtype, int ldr, int og,
                                 const float* w, float eps, void* out, int out_dtype, int T, int H, int m,
                                 hipStream_t stream) {
  GS_REQUIRE(T >= 0 && H > 0 && m > 0 && og >= 0 && og + H * m <= ldr, "memory_outnorm: bad sizes T=%d H=%d m=%d, or a gate outside the rows of %d", T, H, m, ldr);
  GS_REQUIRE(hs >= m && ds > 0, "memory_outnorm: bad strides %d, %d", hs, ds);
  GS_REQUIRE(eps > 0.f, "memory_outnorm: eps must be positive");
  if (T == 0) return 0;
  const int threads = H >= 4 ? 256 : 64 * H;
  if (rows_dtype == GS_F32 && out_dtype == GS_F32)
    memory_outnorm_kernel<float, float><<<T, threads, 0, stream>>>(o, hs, den, ds, gates, (const float*)rows, ldr, og, w, eps, (float*)out, H, m);
  else if (rows_dtype == GS_BF16 && out_dtype == GS_BF16)
    memory_outnorm_kernel<bf16, bf16><<<T, threads, 0, stream>>>(o, hs, den, ds, gates, (const bf16*)rows, ldr, og, w, eps, (bf16*)out, H, m);
  else if (rows_dtype == GS_BF16 && out_dtype == GS_F32)
    memory_outnorm_kernel<bf16, float><<<T, threads, 0, stream>>>(o, hs, den, ds, gates, (const bf16*)rows, ldr, og, w, eps, (float*)out, H, m);
  else if (rows_dtype == GS_F32 && out_dtype == GS_BF16)
    memory_outnorm_kernel<float, bf16><<<T, threads, 0, stream>>>(o, hs, den, ds, gates, (const float*)rows, ldr, og, w, eps, (bf16*)out, H, m);
  else
    GS_REQUIRE(false, "memory_outnorm: unknown dtypes %d %d", rows_dtype, out_dtype);
  GS_LAUNCH_CHECK("memory_outnorm");
  return 0;
}
