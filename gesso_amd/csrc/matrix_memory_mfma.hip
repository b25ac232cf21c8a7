// The matrix memory's recurrence for prompt portions, on the matrix cores (bfloat16 rows).
//
// The same recurrence as gated_recurrence.hip walks token by token with a decay a head, write strengths and a column of
// ones: per sequence and head, S <- a_t S + w_t k_t [v_t | 1]^T, [o_t | d_t] = S^T (q_scale q_t), a_t, w_t <= 1 given as
// base-2 logarithms la, lw.  Taken 32 tokens at a time: with Q, K (32 x n), V (32 x m) the rows of a run, S and the vector
// N (the state's last column) before it, c_t = la_0 + ... + la_t within the run and L its last token,
//
//   O  = diag(2^c_t) Q S + A V,     A[t][s] = (q_t . k_s) 2^(c_t - c_s + lw_s) for s <= t, else 0
//   d  = diag(2^c_t) Q N + A 1
//   S' = 2^c_L S + sum_s 2^(c_L - c_s + lw_s) k_s v_s^T,     N' likewise with k_s alone
//
// Every exponent is at most zero.  One block per (run of tokens, head, 128 value columns), four wavefronts, each owning 32
// of the columns; its slice of the state (n x 32) stays in its accumulators.  Products are v_mfma_f32_32x32x16_bf16.  Q, K
// and V are bfloat16 as their product left them and enter as they are; what is held in 32 bits (A, the state, the weighted
// keys) enters as two bfloat16 terms, the value's rounding and the rounding of what is left; sums are float32.
//
// A and the state never pass through LDS.  A result's lane (column l % 32) holds rows 8 (e / 4) + 4 (l / 32) + e % 4; as
// the operand of the next product its register q of a step of 16 stands for the inner index 8 (q / 4) + 4 (l / 32) + q % 4,
// and the other operand is read in the same order (two 8-byte reads).  A is computed transposed (rows s, columns t), the
// state as rows i, columns j, so that both come out in that form.
//
// N lies in LDS as float32: its products with the queries are shared out between the wavefronts, its increment is a row sum
// of the weighted keys, and both are put in place in the next run between its two barriers.
//
// OUT = false: what a run writes, starting from nothing (B goes to `state`, the product of its decays to `seg_d`); no
// queries, no outputs.  With the chain over segments (gated_state_chain_diagonal) this lets a long portion's segments run
// side by side.
#include "common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 mm_bf16x8_t;
typedef __attribute__((ext_vector_type(4))) __bf16 mm_bf16x4_t;
typedef __attribute__((ext_vector_type(16))) float mm_f32x16_t;
typedef __attribute__((ext_vector_type(4))) unsigned mm_u32x4_t;

constexpr int MM_C = 32;          // tokens a run
constexpr int MM_MTB = 128;       // value columns a block
constexpr int MM_LDT = MM_C + 8;  // elements per LDS row of the transposed operands

template <int NT, bool OUT>
__global__ __launch_bounds__(256) void memory_chunk_kernel(const bf16* __restrict__ x, int ld, int oq, int ok, int ov,
                                                           float q_scale, const float* __restrict__ logs, int ldg,
                                                           float* __restrict__ state, const int* __restrict__ q_start,
                                                           const int* __restrict__ slots, float* __restrict__ out,
                                                           float* __restrict__ den, float* __restrict__ seg_d, int H, int n,
                                                           int m) {
  constexpr int NP = 32 * NT, LDQ = NP + 8;
  extern __shared__ __align__(16) uint16_t mm_lds[];
  uint16_t* KTh = mm_lds;                      // [NP][MM_LDT] each: the weighted keys, transposed
  uint16_t* KTl = KTh + NP * MM_LDT;
  uint16_t* VT = KTl + NP * MM_LDT;            // [MM_MTB][MM_LDT]: values, transposed
  uint16_t* Q = VT + MM_MTB * MM_LDT;          // [MM_C][LDQ] each (with OUT)
  uint16_t* K = Q + MM_C * LDQ;
  __shared__ __align__(16) float nv[NP], ninc[NP];                     // N, and what the run before adds to it
  __shared__ __align__(16) float cl[MM_C], lift[MM_C], grow[MM_C];     // c_t; lw_s - c_s; 2^c_t q_scale
  __shared__ float dpart[4][2][MM_C], rsum[2][MM_C];                   // shares of Q N, row sums of A
  const int seq = blockIdx.x, h = blockIdx.y, j0 = blockIdx.z * MM_MTB;
  const int t0 = q_start[seq], t1 = q_start[seq + 1];
  if (t1 <= t0) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l32 = lane & 31, half = lane >> 5;
  const int jw = wave * 32;
  const bool live = j0 + jw < m;               // a wavefront whose columns all lie beyond m only helps staging
  const bool first_block = blockIdx.z == 0;    // the block that also keeps N
  const int ms = m + 1;                        // a state row's length
  float* S = state + ((size_t)slots[seq] * H + h) * n * ms;

  mm_f32x16_t acc[NT];
#pragma unroll
  for (int it = 0; it < NT; ++it)
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int i = it * 32 + 8 * (e / 4) + 4 * half + e % 4, j = j0 + jw + l32;
      acc[it][e] = (OUT && i < n && j < m) ? S[(size_t)i * ms + j] : 0.f;
    }
  for (int i = tid; i < NP; i += 256) {
    nv[i] = (OUT && i < n) ? S[(size_t)i * ms + m] : 0.f;
    ninc[i] = 0.f;
  }
  float held = 1.f;                            // by what the run before shrinks N
  float total = 0.f;                           // the sum of la over the runs gone by

  // A run's rows come as 16-byte pieces (eight features of one token), asked for while the run before is computed: piece u
  // of a thread is token tid % 32, features 8 (tid / 32 + 8 u) ...; so a lane's pieces all belong to its own token.
  constexpr int UQ = (NP / 8 + 7) / 8, UV = MM_MTB / 64;
  mm_u32x4_t rq[OUT ? UQ : 1], rk[UQ], rv[UV];
  float la = 0.f, lw = 0.f;
  const int pc = tid >> 5;
  auto fetch = [&](int tb, int nb) {
    const bool has = l32 < nb;
    const bf16* row = x + (size_t)(tb + (has ? l32 : 0)) * ld;
#pragma unroll
    for (int u = 0; u < UQ; ++u) {
      const int i = 8 * (pc + 8 * u);
      rk[u] = mm_u32x4_t{0u, 0u, 0u, 0u};
      if constexpr (OUT) rq[u] = mm_u32x4_t{0u, 0u, 0u, 0u};
      if (has && i < n) {
        rk[u] = *reinterpret_cast<const mm_u32x4_t*>(row + ok + h * n + i);
        if constexpr (OUT) rq[u] = *reinterpret_cast<const mm_u32x4_t*>(row + oq + h * n + i);
      }
    }
#pragma unroll
    for (int u = 0; u < UV; ++u) {
      const int c = 8 * (pc + 8 * u);
      rv[u] = mm_u32x4_t{0u, 0u, 0u, 0u};
      if (has && j0 + c < m) rv[u] = *reinterpret_cast<const mm_u32x4_t*>(row + ov + h * m + j0 + c);
    }
    const float* g = logs + (size_t)(tb + (has ? l32 : 0)) * ldg + h;
    la = has ? g[0] : 0.f;
    lw = has ? g[H] : 0.f;
  };
  auto store_den = [&](int tb, int nb) {        // the run before's d, from its shares (32 lanes)
    if (OUT && first_block && tid < nb) {
      float s = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) s += dpart[w][0][tid] + dpart[w][1][tid];
      den[(size_t)(tb + tid) * H + h] = s * grow[tid] + q_scale * (rsum[0][tid] + rsum[1][tid]);
    }
  };
  fetch(t0, t1 - t0 < MM_C ? t1 - t0 : MM_C);
  for (int tb = t0; tb < t1; tb += MM_C) {
    const int nb = t1 - tb < MM_C ? t1 - tb : MM_C;
    __syncthreads();                            // the run before has been read, its shares are in place
    if (tb > t0) store_den(tb - MM_C, MM_C);
    if (first_block)
      for (int i = tid; i < NP; i += 256) nv[i] = held * nv[i] + ninc[i];
    if (OUT) __syncthreads();                   // (grow has been read)
    // c_t: the inclusive sum over this lane's 32 tokens; every wavefront makes its own (both halves hold the same)
    float c = la;
#pragma unroll
    for (int o = 1; o < 32; o <<= 1) {
      const float up = __shfl_up(c, o, 32);
      if (l32 >= o) c += up;
    }
    const float last = __shfl(c, 31, 32);       // (tokens beyond the run's end have la = 0)
    const float weight = l32 < nb ? __builtin_amdgcn_exp2f(last - c + lw) : 0.f;
    if (OUT && tid < MM_C) {
      cl[tid] = c;
      lift[tid] = lw - c;
      grow[tid] = __builtin_amdgcn_exp2f(c) * q_scale;
    }
#pragma unroll
    for (int u = 0; u < UQ; ++u) {
      const int i = 8 * (pc + 8 * u);
      if (i < NP) {
        if constexpr (OUT) {
          *reinterpret_cast<mm_u32x4_t*>(Q + l32 * LDQ + i) = rq[u];
          *reinterpret_cast<mm_u32x4_t*>(K + l32 * LDQ + i) = rk[u];
        }
        const unsigned w4[4] = {rk[u].x, rk[u].y, rk[u].z, rk[u].w};
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float kv = __uint_as_float(e & 1 ? w4[e / 2] & 0xffff0000u : w4[e / 2] << 16) * weight;
          const bf16 hi = f32_to_bf16(kv);
          KTh[(i + e) * MM_LDT + l32] = hi.x;
          KTl[(i + e) * MM_LDT + l32] = f32_to_bf16(kv - to_f32(hi)).x;
        }
      }
    }
#pragma unroll
    for (int u = 0; u < UV; ++u) {
      const int cc = 8 * (pc + 8 * u);
      const unsigned w4[4] = {rv[u].x, rv[u].y, rv[u].z, rv[u].w};
#pragma unroll
      for (int e = 0; e < 8; ++e) VT[(cc + e) * MM_LDT + l32] = (uint16_t)(e & 1 ? w4[e / 2] >> 16 : w4[e / 2] & 0xffffu);
    }
    __syncthreads();
    if (tb + MM_C < t1) fetch(tb + MM_C, t1 - tb - MM_C < MM_C ? t1 - tb - MM_C : MM_C);   // the next run's rows, meanwhile
    held = __builtin_amdgcn_exp2f(last);
    total += last;
    if (first_block) {
      for (int i = tid; i < NP; i += 256) {     // the row sums of the weighted keys
        float s = 0.f;
#pragma unroll
        for (int g8 = 0; g8 < MM_C / 8; ++g8) {
          const mm_bf16x8_t a = *reinterpret_cast<const mm_bf16x8_t*>(KTh + i * MM_LDT + 8 * g8);
          const mm_bf16x8_t b = *reinterpret_cast<const mm_bf16x8_t*>(KTl + i * MM_LDT + 8 * g8);
#pragma unroll
          for (int e = 0; e < 8; ++e) s += (float)a[e] + (float)b[e];
        }
        ninc[i] = s;
      }
      if constexpr (OUT) {
        // this wavefront's quarter of the features of q_t . N, a half of it a lane
        float s = 0.f;
#pragma unroll
        for (int g8 = 0; g8 < (NP / 8 + 7) / 8; ++g8) {
          const int i = 8 * (2 * (wave + 4 * g8) + half);
          if (i < NP) {
            const mm_bf16x8_t q8 = *reinterpret_cast<const mm_bf16x8_t*>(Q + l32 * LDQ + i);
#pragma unroll
            for (int e = 0; e < 8; ++e) s = fmaf((float)q8[e], nv[i + e], s);
          }
        }
        dpart[wave][half][l32] = s;
      }
    }
    if (!live) continue;                        // (the first block's first wavefront always has columns)

    if constexpr (OUT) {
      mm_f32x16_t at;                           // q_t . k_s: rows s, column t
#pragma unroll
      for (int e = 0; e < 16; ++e) at[e] = 0.f;
      const int ro = l32 * LDQ + half * 8;
#pragma unroll
      for (int ks = 0; ks < NP / 16; ++ks)
        at = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const mm_bf16x8_t*>(K + ro + ks * 16),
                                                     *reinterpret_cast<const mm_bf16x8_t*>(Q + ro + ks * 16), at, 0, 0, 0);
      // what the state before the run gives: rows t, columns j (two accumulators in turn)
      mm_f32x16_t o, ob;
#pragma unroll
      for (int e = 0; e < 16; ++e) o[e] = ob[e] = 0.f;
#pragma unroll
      for (int ks = 0; ks < NP / 16; ++ks) {
        const uint16_t* qp = Q + l32 * LDQ + 16 * ks + 4 * half;
        const mm_bf16x4_t q0 = *reinterpret_cast<const mm_bf16x4_t*>(qp), q1 = *reinterpret_cast<const mm_bf16x4_t*>(qp + 8);
        mm_bf16x8_t q8, sh, sl;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          q8[e] = q0[e];
          q8[4 + e] = q1[e];
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float v = acc[ks / 2][8 * (ks % 2) + e];
          const __bf16 hi = (__bf16)v;
          sh[e] = hi;
          sl[e] = (__bf16)(v - (float)hi);
        }
        o = __builtin_amdgcn_mfma_f32_32x32x16_bf16(q8, sh, o, 0, 0, 0);
        ob = __builtin_amdgcn_mfma_f32_32x32x16_bf16(q8, sl, ob, 0, 0, 0);
      }
      // A: the causal rule, the decay between the two and the write strength; as operands of the next product
      const float ct = cl[l32];
      mm_bf16x8_t ah[2], al[2];
      float rs = 0.f;
#pragma unroll
      for (int g4 = 0; g4 < 4; ++g4) {
        const float4 lf = *reinterpret_cast<const float4*>(&lift[8 * g4 + 4 * half]);
        const float l4[4] = {lf.x, lf.y, lf.z, lf.w};
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          const int s = 8 * g4 + 4 * half + q, e = 4 * g4 + q;
          const float a = s <= l32 ? at[e] * __builtin_amdgcn_exp2f(ct + l4[q]) : 0.f;
          rs += a;
          const __bf16 hi = (__bf16)a;
          ah[e / 8][e % 8] = hi;
          al[e / 8][e % 8] = (__bf16)(a - (float)hi);
        }
      }
      if (first_block && wave == 0) rsum[half][l32] = rs;
      {
        mm_f32x16_t p;
#pragma unroll
        for (int e = 0; e < 16; ++e) p[e] = 0.f;
        const int vo = (jw + l32) * MM_LDT;
#pragma unroll
        for (int k2 = 0; k2 < 2; ++k2) {
          const mm_bf16x4_t v0 = *reinterpret_cast<const mm_bf16x4_t*>(VT + vo + 16 * k2 + 4 * half);
          const mm_bf16x4_t v1 = *reinterpret_cast<const mm_bf16x4_t*>(VT + vo + 16 * k2 + 8 + 4 * half);
          mm_bf16x8_t v8;
#pragma unroll
          for (int q = 0; q < 4; ++q) {
            v8[q] = v0[q];
            v8[4 + q] = v1[q];
          }
          p = __builtin_amdgcn_mfma_f32_32x32x16_bf16(ah[k2], v8, p, 0, 0, 0);
          p = __builtin_amdgcn_mfma_f32_32x32x16_bf16(al[k2], v8, p, 0, 0, 0);
        }
        const int j = j0 + jw + l32;
#pragma unroll
        for (int g4 = 0; g4 < 4; ++g4) {
          const float4 gr = *reinterpret_cast<const float4*>(&grow[8 * g4 + 4 * half]);
          const float g[4] = {gr.x, gr.y, gr.z, gr.w};
#pragma unroll
          for (int q = 0; q < 4; ++q) {
            const int t = 8 * g4 + 4 * half + q, e = 4 * g4 + q;
            if (j < m && t < nb) out[((size_t)(tb + t) * H + h) * m + j] = fmaf(o[e] + ob[e], g[q], q_scale * p[e]);
          }
        }
      }
    }
    // the state after the run: rows i, columns j
#pragma unroll
    for (int it = 0; it < NT; ++it) {
#pragma unroll
      for (int e = 0; e < 16; ++e) acc[it][e] *= held;
#pragma unroll
      for (int k2 = 0; k2 < 2; ++k2) {
        const mm_bf16x8_t v8 = *reinterpret_cast<const mm_bf16x8_t*>(VT + (jw + l32) * MM_LDT + 16 * k2 + 8 * half);
        const int ko = (it * 32 + l32) * MM_LDT + 16 * k2 + 8 * half;
        acc[it] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const mm_bf16x8_t*>(KTh + ko), v8, acc[it], 0, 0, 0);
        acc[it] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const mm_bf16x8_t*>(KTl + ko), v8, acc[it], 0, 0, 0);
      }
    }
  }
  __syncthreads();
  const int tail = (t1 - t0 - 1) / MM_C * MM_C;
  store_den(t0 + tail, t1 - t0 - tail);
  if (first_block)
    for (int i = tid; i < n; i += 256) {
      S[(size_t)i * ms + m] = held * nv[i] + ninc[i];
      if (!OUT) seg_d[((size_t)slots[seq] * H + h) * n + i] = __builtin_amdgcn_exp2f(total);
    }
#pragma unroll
  for (int it = 0; it < NT; ++it)
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int i = it * 32 + 8 * (e / 4) + 4 * half + e % 4, j = j0 + jw + l32;
      if (i < n && j < m) S[(size_t)i * ms + j] = acc[it][e];
    }
}

template <int NT, bool OUT>
static int mm_launch(dim3 grid, hipStream_t stream, const bf16* x, int ld, int oq, int ok, int ov, float q_scale,
                     const float* logs, int ldg, float* state, const int* q_start, const int* slots, float* out, float* den,
                     float* seg_d, int H, int n, int m) {
  constexpr int NP = 32 * NT, LDQ = NP + 8;
  const size_t lds = (size_t)(2 * NP * MM_LDT + MM_MTB * MM_LDT + (OUT ? 2 * MM_C * LDQ : 0)) * sizeof(uint16_t);
  // more than the default limit of dynamic LDS for wide keys: asked for once per kernel
  static const hipError_t asked = hipFuncSetAttribute(reinterpret_cast<const void*>(&memory_chunk_kernel<NT, OUT>),
                                                      hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  GS_REQUIRE(asked == hipSuccess, "memory_chunks: cannot raise the LDS limit: %s", hipGetErrorString(asked));
  memory_chunk_kernel<NT, OUT><<<grid, 256, lds, stream>>>(x, ld, oq, ok, ov, q_scale, logs, ldg, state, q_start, slots, out,
                                                           den, seg_d, H, n, m);
  return 0;
}

// Whether the kernel takes these rows: keys up to 256 wide, every 16-byte piece whole and aligned.
extern "C" int gs_memory_chunks_supports(int n, int m, int ld, int oq, int ok, int ov) {
  return n > 0 && n <= 256 && n % 8 == 0 && m > 0 && m % 8 == 0 && ld % 8 == 0 && oq % 8 == 0 && ok % 8 == 0 && ov % 8 == 0;
}

// x (T, ld) bfloat16 rows; logs (T, ldg) float32: la of head h at [h], lw at [H + h]; state (slots, H, n, m + 1).  With out
// (T, H m) and den (T, H): from the state, advanced.  With seg_d (slots, H, n) instead: from nothing, B left in state.
extern "C" int gs_memory_chunks(const void* x, int ld, int oq, int ok, int ov, float q_scale, const float* logs, int ldg,
                                float* state, const int* q_start, const int* slots, float* out, float* den, float* seg_d,
                                int nseq, int H, int n, int m, hipStream_t stream) {
  GS_REQUIRE(nseq >= 0 && H > 0 && H <= 65535 && gs_memory_chunks_supports(n, m, ld, oq, ok, ov) && ((uintptr_t)x & 15) == 0,
             "memory_chunks: sizes nseq=%d H=%d n=%d m=%d or rows of %d are not taken", nseq, H, n, m, ld);
  GS_REQUIRE(oq >= 0 && ok >= 0 && ov >= 0 && oq + H * n <= ld && ok + H * n <= ld && ov + H * m <= ld,
             "memory_chunks: q, k or v lie outside the rows of %d", ld);
  GS_REQUIRE(ldg >= 2 * H, "memory_chunks: the gates lie outside their rows of %d", ldg);
  GS_REQUIRE((out != nullptr) == (den != nullptr) && (out != nullptr) != (seg_d != nullptr),
             "memory_chunks: outputs with their denominators, or what the runs do to a state");
  if (nseq == 0) return 0;
  dim3 grid(nseq, H, (m + MM_MTB - 1) / MM_MTB);
  GS_REQUIRE(grid.z <= 65535, "memory_chunks: too many value columns");
  int rc = 0;
#define MM_RUN(NT)                                                                                                          \
  rc = out ? mm_launch<NT, true>(grid, stream, (const bf16*)x, ld, oq, ok, ov, q_scale, logs, ldg, state, q_start, slots,   \
                                 out, den, seg_d, H, n, m)                                                                  \
           : mm_launch<NT, false>(grid, stream, (const bf16*)x, ld, oq, ok, ov, q_scale, logs, ldg, state, q_start, slots,  \
                                  out, den, seg_d, H, n, m)
  if (n <= 32) MM_RUN(1);
  else if (n <= 64) MM_RUN(2);
  else if (n <= 128) MM_RUN(4);
  else MM_RUN(8);
#undef MM_RUN
  if (rc != 0) return rc;
  GS_LAUNCH_CHECK("memory_chunks");
  return 0;
}
