// The kernels of decode attention: one query token per sequence over its paged keys and values, bfloat16 cache
// (attention_decode.hip describes them; attention_decode_maps.hip launches the form for two maps a head).
#pragma once
#include "common.h"

#define DEC_MAXG 8
#define DEC_LOG2E 1.4426950408889634f

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;

// With RAW, q points at rows of q|k|v as their product left them (q heads, then k heads, then v heads), and the
// kernel does what comes between that product and attention itself: the head norms of q and k, the rotation, and
// the write of the new key and value into their page.  Every block norms and rotates its own queries; the block
// whose keys end with the new one norms and rotates it, keeps it and the value in LDS for its scores, and writes
// both to the cache for the steps to come.  Heads of 64 or 128, rotated whole.
// Where column c of sequence seq's output goes: a row of `width`, or tiled rows (out_tiles = ceil(nseq / 16) > 0),
// the order in which the product that follows takes them.
__device__ __forceinline__ size_t out_index(int seq, int c, int width, int out_tiles) {
  return out_tiles ? tiled_index(seq, c, out_tiles) : (size_t)seq * width + c;
}

struct DecodeRaw {
  const float* qw;       // (D) head norm weights, or null for no norm
  const float* kw;
  float eps;
  const float* cos_t;    // (positions, D / 2)
  const float* sin_t;
  int write_kv;          // 0: another layer owns the cache; the new key is already in it
  // (read with and without RAW) chunk > 0: the query sees no key before the first position of its own run of `chunk`
  // positions; sink: one more term exp(0), without a value, in the softmax's denominator
  int chunk;
  int sink;
  // softcap > 0: a score becomes softcap tanh(score / softcap).  keep_first > 0 (with a window, without runs): the
  // sequence's first keep_first positions stay visible when the window has passed them.  sinks (one float32 a head):
  // the extra term of the denominator is exp(sinks[h]) instead of exp(0).
  float softcap;
  int keep_first;
  const float* sinks;
};

// MAPS = 2: attention as the difference of two softmax maps over one value row (attention_maps.hip has the definition).
// D is then a cached key row, a head's two keys of D / 2 features side by side, and the G columns are the 2 maps of G / 2
// query heads: column r16 holds head r16 / 2's query of map r16 % 2 beside zeros in the other map's features, so that one
// product over the whole key row gives every column its own map's score.  Values are DV wide.  Once the wavefronts (or the
// splits) are merged, the maps' difference is normed, gated and stored.  Groups of more than G / 2 query heads are cut into
// `parts` blocks.
struct DecodeMaps {
  float lam, eps, out_scale;
  int gate_col;          // the column of the query's row where the heads' gates stand (< 0: none)
  int parts;
};

// One query head's end, by one wavefront: o = o1 - lam o2 (both in LDS, divided by their sums), normed, gated, stored at dst.
template <int DV>
__device__ __forceinline__ void finish_maps(const float* o1, const float* o2, const DecodeMaps& dm, float gate, bf16* dst,
                                            int lane) {
  constexpr int NV = (DV + 63) / 64;
  float o[NV], ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int j = lane + 64 * i;
    o[i] = j < DV ? o1[j] - dm.lam * o2[j] : 0.f;
    ss += o[i] * o[i];
  }
  const float f = norm_inverse(wave_sum_dpp(ss), (float)DV, dm.eps) * dm.out_scale * gate;
#pragma unroll
  for (int i = 0; i < NV; ++i)
    if (lane + 64 * i < DV) dst[lane + 64 * i] = f32_to_bf16(o[i] * f);
}

template <int D, int G, int W, int RAW, int DV = D, int MAPS = 1>
__global__ __launch_bounds__(W * 64) void attention_decode_kernel(
    const bf16* __restrict__ q, int q_stride, bf16* kcache, bf16* vcache,
    const int* __restrict__ positions, const int* __restrict__ block_table, int max_blocks, int page_size,
    unsigned page_magic, int window, float scale, bf16* __restrict__ out, float* __restrict__ part_o,
    float* __restrict__ part_ml, int nh, int nkv, int out_tiles, DecodeRaw raw, DecodeMaps dm) {
  static_assert(MAPS == 1 ? DV == D : (MAPS == 2 && !RAW && G % 2 == 0), "values of another width and two maps go together");
  static_assert(!RAW || D == 64 || D == 128, "the fused head norm and rotation are written for heads of 64 and 128");
  constexpr int DC = DV / 8;              // 16-byte chunks per value row
  constexpr int DL = DC <= 2 ? 2 : DC <= 4 ? 4 : DC <= 8 ? 8 : DC <= 16 ? 16 : DC <= 32 ? 32 : 64;   // lanes a value row: a power of two (those beyond DC idle)
  constexpr int KG = 64 / DL;             // key groups per wavefront in the value phase
  constexpr int NI = 64 / KG;             // keys per lane in the value phase
  constexpr int KS = (D + 31) / 32;       // steps of 32 features in the score products
  static_assert(D % 8 == 0 && DV % 8 == 0 && DC >= 2 && DC <= 64 && G <= 16, "head widths are multiples of 8 from 16 to 512");
  // What the registers allow (256 a lane at eight wavefronts a block): the next tile's rows in flight while
  // this one is computed, for rows of up to 64.
  constexpr bool PIPE = D <= 64 && DV <= 64;
  __shared__ float ps[W][G][64];          // a tile's probabilities, then read per key in the value phase
  __shared__ float al[W][G];              // by how much a tile shrinks what was accumulated before it
  __shared__ float wm[W][G], wl[W][G];
  __shared__ float wacc[W][G][DV];

  const int split = blockIdx.x, nsplit = gridDim.x, kvh = blockIdx.y, seq = blockIdx.z;
  const int kvc = MAPS == 1 ? kvh : kvh / dm.parts, nkc = MAPS == 1 ? nkv : nkv / dm.parts;   // the cache's key head, and their number
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int r16 = lane & 15, kg = lane >> 4;
  const int pos = positions[seq];
  int lo_real = window > 0 ? (pos - window + 1 > 0 ? pos - window + 1 : 0) : 0;
  if (raw.chunk > 0 && pos - pos % raw.chunk > lo_real) lo_real = pos - pos % raw.chunk;
  // The kept first positions that the window has passed stand before the window's keys in one row of places: place
  // lo + i is key i for the `kept` first places, and key lo + i (itself) from there on.
  const int kept = (raw.keep_first > 0 && window > 0 && raw.chunk == 0) ? (raw.keep_first < lo_real ? raw.keep_first : lo_real) : 0;
  const int lo = lo_real - kept;
  const int nkeys = pos - lo + 1;
  // this block's share of the keys, in whole tiles of 64
  const int tiles = (nkeys + 63) >> 6;
  const int tper = (tiles + nsplit - 1) / nsplit;
  const int t0 = split * tper, t1 = (t0 + tper < tiles) ? t0 + tper : tiles;
  const int* bt = block_table + (size_t)seq * max_blocks;
  const int kq = lane / DL;
  const bool dlive = DL == DC || lane % DL < DC;       // (a spare lane loads and sums what its neighbours do, and stores nothing)
  const int dc = dlive ? lane % DL : DC - 1;

  // which row of the caches is key u's (u <= pos)
  // (u / page_size as one multiplication, page_magic = floor(2^32 / page_size) + 1, exact while u page_size < 2^32:
  // no branch near the loads, which would make the compiler wait for every load in flight)
  auto row_off = [&](int u) -> long {
    u = u < lo_real ? u - lo : u;          // a place before the window's first key holds a kept first position
    const int pg = (int)__umulhi((unsigned)u, page_magic);
    const int r = u - pg * page_size;
    return ((long)bt[pg] * nkc + kvc) * page_size + r;
  };
  // The loads of tile t.  Keys, as the first operand of the score products: lane (r16, kg) holds, of the four
  // keys 4 r16 + kt, features 32 s + 8 kg .. + 8.  Values: the lane's chunk of eight features of the value rows
  // of its NI keys.  Keys beyond pos are read from key pos (they are masked, their probabilities are zero).
  auto issue = [&](int t, bf16x8_t (*kreg)[KS], uint4* vreg) {
    const int base = lo + (t << 6);
    long ko[4], vo[NI];
#pragma unroll
    for (int kt = 0; kt < 4; ++kt) {
      const int u = base + 4 * r16 + kt;
      ko[kt] = row_off(u <= pos ? u : pos) * D + kg * 8;
    }
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int uu = base + kq + i * KG;
      vo[i] = row_off(uu <= pos ? uu : pos) * DV + dc * 8;
    }
#pragma unroll
    for (int kt = 0; kt < 4; ++kt)
#pragma unroll
      for (int st = 0; st < KS; ++st) {
        if (32 * st + 8 * kg < D)
          kreg[kt][st] = *reinterpret_cast<const bf16x8_t*>(kcache + ko[kt] + 32 * st);
        else
          kreg[kt][st] = bf16x8_t{0, 0, 0, 0, 0, 0, 0, 0};
      }
#pragma unroll
    for (int i = 0; i < NI; ++i) vreg[i] = *reinterpret_cast<const uint4*>(vcache + vo[i]);
  };

  // Loads in the order of what they wait for: the queries, the norm weights and the step's own key and value
  // (they wait for nothing), the rotation factors and the page numbers (for the position), the key and value rows
  // (for the page numbers).  Loads return in order, so the queries are normed and rotated while the rows are on
  // their way.
  // the queries as the second operand: lane (r16, kg) holds head r16's features 32 s + 8 kg .. + 8
  // (lanes past the group load head 0's: every lane loads, no branch hides a load from the compiler's count)
  bf16x8_t qreg[KS];
#pragma unroll
  for (int st = 0; st < KS; ++st) {
    if constexpr (MAPS == 2) {
      const int f0 = 32 * st + 8 * kg, map = f0 / (D / 2);
      qreg[st] = *reinterpret_cast<const bf16x8_t*>(q + (size_t)seq * q_stride + (size_t)(kvh * G + (r16 < G ? r16 : 0)) * (D / 2) + (f0 < D ? f0 - map * (D / 2) : 0));
      if (r16 >= G || map != (r16 & 1)) qreg[st] = bf16x8_t{0, 0, 0, 0, 0, 0, 0, 0};
    } else if (32 * st + 8 * kg < D)
      qreg[st] = *reinterpret_cast<const bf16x8_t*>(q + (size_t)seq * q_stride + (size_t)(kvh * G + (r16 < G ? r16 : 0)) * D + 32 * st + 8 * kg);
    else
      qreg[st] = bf16x8_t{0, 0, 0, 0, 0, 0, 0, 0};
    if (!RAW && r16 >= G) qreg[st] = bf16x8_t{0, 0, 0, 0, 0, 0, 0, 0};
  }
  // Every wavefront keeps a copy of its own of the step's key and value in LDS (the wavefront whose tile holds the
  // new key reads them there: the cache's rows were loaded before they were written), so no wavefront waits for
  // another; wavefront 0 of the block whose keys end with the new one also writes them to the cache.
  __shared__ __align__(16) uint16_t knew[RAW ? W : 1][RAW ? D : 8], vnew[RAW ? W : 1][RAW ? D : 8];
  const bool has_new = RAW && raw.write_kv && t0 < t1 && t1 == tiles;   // this block's keys end with the new one
  constexpr int E = D >= 64 ? D / 64 : 1;
  float qw8[RAW ? KS : 1][8], c8[RAW ? KS / 2 : 1][8], s8[RAW ? KS / 2 : 1][8];
  float kraw_f[E], kw_f[E], kc_f = 1.f, ks_f = 0.f;
  bf16 vraw_b[E];
  if constexpr (RAW != 0) {
    if (raw.qw) {
#pragma unroll
      for (int st = 0; st < KS; ++st) load8f(raw.qw + 32 * st + 8 * kg, qw8[st]);
    }
    const bf16* kraw = q + (size_t)seq * q_stride + (size_t)(nh + kvh) * D;
    const bf16* vraw = q + (size_t)seq * q_stride + (size_t)(nh + nkv + kvh) * D;
#pragma unroll
    for (int e = 0; e < E; ++e) {
      kraw_f[e] = to_f32(kraw[lane + 64 * e]);
      vraw_b[e] = vraw[lane + 64 * e];
      kw_f[e] = raw.kw ? raw.kw[lane + 64 * e] : 1.f;
    }
    // (weights and rotation factors in 16-byte loads: the tables' rows and this lane's offsets are multiples of 8)
#pragma unroll
    for (int st = 0; st < KS / 2; ++st) {
      load8f(raw.cos_t + (size_t)pos * (D / 2) + 32 * st + 8 * kg, c8[st]);
      load8f(raw.sin_t + (size_t)pos * (D / 2) + 32 * st + 8 * kg, s8[st]);
    }
    const int pi = E == 2 ? lane : (lane & 31);          // index of this lane's pair of the key
    kc_f = raw.cos_t[(size_t)pos * (D / 2) + pi];
    ks_f = raw.sin_t[(size_t)pos * (D / 2) + pi];
  }
  bf16x8_t kn[4][KS];
  uint4 vn[NI];
  int t = t0 + wave;
  // (a wavefront without a tile asks for the block's first one: its address is a valid one, and a load behind a
  // branch would make the compiler wait for every load in flight where it needs the queries)
  issue(t < t1 ? t : (t0 < tiles ? t0 : 0), kn, vn);

  if constexpr (RAW != 0) {
    // head norm and rotation of this lane's part of its query: float32 arithmetic on the product's bfloat16
    // values, rounded to bfloat16 again, as the separate kernel does.  The halves of a rotation pair (i, i + D/2)
    // are steps KS/2 apart in the same lane.
    float qf[KS][8];
    float ss = 0.f;
#pragma unroll
    for (int st = 0; st < KS; ++st)
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        qf[st][j] = (float)qreg[st][j];
        ss += qf[st][j] * qf[st][j];
      }
    if (raw.qw) {
      const float inv = norm_inverse(group4_sum(ss), (float)D, raw.eps);
#pragma unroll
      for (int st = 0; st < KS; ++st)
#pragma unroll
        for (int j = 0; j < 8; ++j) qf[st][j] = qf[st][j] * inv * qw8[st][j];
    }
#pragma unroll
    for (int st = 0; st < KS / 2; ++st)
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float a = qf[st][j], b = qf[st + KS / 2][j];
        qf[st][j] = a * c8[st][j] - b * s8[st][j];
        qf[st + KS / 2][j] = a * s8[st][j] + b * c8[st][j];
      }
#pragma unroll
    for (int st = 0; st < KS; ++st)
#pragma unroll
      for (int j = 0; j < 8; ++j) qreg[st][j] = (r16 < G) ? (__bf16)qf[st][j] : (__bf16)0.f;
    // the new key and value: lane = feature (and feature + 64 for heads of 128)
    if (raw.write_kv) {
      float kf[E];
      float ks = 0.f;
#pragma unroll
      for (int e = 0; e < E; ++e) {
        kf[e] = kraw_f[e];
        ks += kf[e] * kf[e];
      }
      if (raw.kw) {
        const float inv = norm_inverse(wave_sum_dpp(ks), (float)D, raw.eps);
#pragma unroll
        for (int e = 0; e < E; ++e) kf[e] = kf[e] * inv * kw_f[e];
      }
      if (E == 2) {
        const float a = kf[0], b = kf[E - 1];
        kf[0] = a * kc_f - b * ks_f;
        kf[E - 1] = a * ks_f + b * kc_f;
      } else {
        const float other = __shfl_xor(kf[0], 32, 64);
        kf[0] = lane < 32 ? kf[0] * kc_f - other * ks_f : other * ks_f + kf[0] * kc_f;
      }
      const long row = row_off(pos) * D;
#pragma unroll
      for (int e = 0; e < E; ++e) {
        const bf16 kb = f32_to_bf16(kf[e]);
        knew[wave][lane + 64 * e] = kb.x;
        vnew[wave][lane + 64 * e] = vraw_b[e].x;
        if (has_new && wave == 0) {
          kcache[row + lane + 64 * e] = kb;
          vcache[row + lane + 64 * e] = vraw_b[e];
        }
      }
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_s_waitcnt(0xc07f);  // LDS writes of this wavefront are visible to its own lanes
    }
  }
  const float qscale = scale * DEC_LOG2E;   // scores are scaled after the product, in float32

  // lanes r16 < G keep the running maximum and sum of head r16; every lane keeps its share of all heads' sums
  float m = -INFINITY, l = 0.f;
  float acc[G][8];
#pragma unroll
  for (int g = 0; g < G; ++g)
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[g][j] = 0.f;

  // one tile: scores, online softmax, values
  auto compute = [&](int t, bf16x8_t (*kc)[KS], uint4* vc) {
    const int base = lo + (t << 6);
    if (RAW && has_new && t == tiles - 1) {
      // the new key's row and the new value's row come from LDS: the cache's rows were loaded before they were written.
      // So do the places past it, which were loaded from the same row of the cache: their probabilities are zero, but
      // what that row held before this step (anything: the page may have been another request's) must not meet them
      const int rel = pos - base;
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
        if (4 * r16 + kt >= rel) {
#pragma unroll
          for (int st = 0; st < KS; ++st) kc[kt][st] = *reinterpret_cast<const bf16x8_t*>(&knew[wave][32 * st + 8 * kg]);
        }
#pragma unroll
      for (int i = 0; i < NI; ++i)
        if (kq + i * KG >= rel) vc[i] = *reinterpret_cast<const uint4*>(&vnew[wave][dc * 8]);
    }
    // sc[kt][i]: head r16, key base + 4 (4 kg + i) + kt
    f32x4_t sc[4];
#pragma unroll
    for (int kt = 0; kt < 4; ++kt) {
      sc[kt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int st = 0; st < KS; ++st) sc[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kc[kt][st], qreg[st], sc[kt], 0, 0, 0);
    }
    float mx = -INFINITY;
#pragma unroll
    for (int kt = 0; kt < 4; ++kt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const bool valid = base + 4 * (4 * kg + i) + kt <= pos;
        float sv = sc[kt][i] * qscale;
        if (raw.softcap > 0.f) {
          // cap tanh(x / cap) = cap (1 - 2 / (1 + e^(2 x / cap))), in the base-2 units the scores are held in
          const float e2 = __builtin_amdgcn_exp2f(sv * (2.f / raw.softcap));
          sv = raw.softcap * DEC_LOG2E * (1.f - 2.f * __builtin_amdgcn_rcpf(1.f + e2));
        }
        sc[kt][i] = valid ? sv : -INFINITY;
        mx = fmaxf(mx, sc[kt][i]);
      }
    const float mn = fmaxf(m, group4_max(mx));   // finite: a tile holds at least one key
    float sum = 0.f;
#pragma unroll
    for (int kt = 0; kt < 4; ++kt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        sc[kt][i] = __builtin_amdgcn_exp2f(sc[kt][i] - mn);   // 0 for masked keys
        sum += sc[kt][i];
      }
    const float alpha = __builtin_amdgcn_exp2f(m - mn);
    l = l * alpha + group4_sum(sum);
    m = mn;
    if (r16 < G) {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        *reinterpret_cast<f32x4_t*>(&ps[wave][r16][4 * (4 * kg + i)]) = f32x4_t{sc[0][i], sc[1][i], sc[2][i], sc[3][i]};
      if (kg == 0) al[wave][r16] = alpha;
    }
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_s_waitcnt(0xc07f);  // LDS writes of this wavefront are visible to its own lanes
#pragma unroll
    for (int g = 0; g < G; ++g) {
      const float a = al[wave][g];
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[g][j] *= a;
    }
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const uint32_t ww[4] = {vc[i].x, vc[i].y, vc[i].z, vc[i].w};
      float v[8];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        v[2 * e] = __uint_as_float(ww[e] << 16);
        v[2 * e + 1] = __uint_as_float(ww[e] & 0xffff0000u);
      }
#pragma unroll
      for (int g = 0; g < G; ++g) {
        const float p = ps[wave][g][kq + i * KG];
#pragma unroll
        for (int j = 0; j < 8; ++j) acc[g][j] += p * v[j];
      }
    }
    __builtin_amdgcn_wave_barrier();
  };

  if (PIPE) {
    // the next tile's loads are in flight while this one is computed: two sets of row registers
    for (; t < t1; t += W) {
      bf16x8_t kc[4][KS];
      uint4 vc[NI];
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int st = 0; st < KS; ++st) kc[kt][st] = kn[kt][st];
#pragma unroll
      for (int i = 0; i < NI; ++i) vc[i] = vn[i];
      if (t + W < t1) issue(t + W, kn, vn);
      compute(t, kc, vc);
    }
  } else {
    // one set of row registers: the first tile's loads were issued above
    if (t < t1) {
      compute(t, kn, vn);
      t += W;
    }
    for (; t < t1; t += W) {
      issue(t, kn, vn);
      compute(t, kn, vn);
    }
  }
  // key groups of a wavefront hold partial sums over different keys for the same features: add them
#pragma unroll
  for (int g = 0; g < G; ++g)
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      float v = acc[g][j];
      for (int o = DL; o < 64; o <<= 1) v += __shfl_xor(v, o, 64);
      acc[g][j] = v;
    }
  if (kq == 0 && dlive) {
#pragma unroll
    for (int g = 0; g < G; ++g)
#pragma unroll
      for (int j = 0; j < 8; ++j) wacc[wave][g][dc * 8 + j] = acc[g][j];
  }
  if (lane < G) {
    wm[wave][lane] = m;
    wl[wave][lane] = l;
  }
  __syncthreads();

  // merge the wavefronts, in wavefront order
  const size_t unit = ((size_t)seq * nkv + kvh) * nsplit + split;  // this block's partial
  for (int i = tid; i < G * DV; i += blockDim.x) {
    int g = i / DV, j = i - g * DV;
    float M = -INFINITY;
    for (int w = 0; w < W; ++w) M = fmaxf(M, wm[w][g]);
    float o = 0.f, L = 0.f;
    if (M > -INFINITY)
      for (int w = 0; w < W; ++w)
        if (wm[w][g] > -INFINITY) {
          float f = __builtin_amdgcn_exp2f(wm[w][g] - M);
          o += wacc[w][g][j] * f;
          L += wl[w][g] * f;
        }
    if (MAPS == 2 && nsplit == 1) {
      wacc[0][g][j] = o / L;                // (nobody else reads this place)
    } else if (nsplit == 1) {
      // (a sink's score is 0; the maxima are in base-2 units of the scaled scores)
      if (raw.sink || raw.sinks)
        L += M > -INFINITY ? __builtin_amdgcn_exp2f((raw.sinks ? raw.sinks[kvh * G + g] * DEC_LOG2E : 0.f) - M) : 1.f;
      out[out_index(seq, (kvh * G + g) * DV + j, nh * DV, out_tiles)] = f32_to_bf16(o / L);
    } else {
      part_o[(unit * G + g) * DV + j] = o;
      if (j == 0) {
        part_ml[(unit * G + g) * 2] = M;
        part_ml[(unit * G + g) * 2 + 1] = L;
      }
    }
  }
  if constexpr (MAPS == 2) {
    if (nsplit > 1) return;
    __syncthreads();
    for (int hq = wave; hq < G / 2; hq += W) {
      const int h = kvh * (G / 2) + hq;
      const float gate = dm.gate_col >= 0 ? 1.f / (1.f + expf(-to_f32(q[(size_t)seq * q_stride + dm.gate_col + h]))) : 1.f;
      finish_maps<DV>(wacc[0][2 * hq], wacc[0][2 * hq + 1], dm, gate, out + ((size_t)seq * (nh / 2) + h) * DV, lane);
    }
  }
}

#define DEC_MAXSPLIT 64

// The splits of two maps, in split order: after the merge each query head's difference is normed, gated and stored.  One block per (sequence,
// group of G maps).
template <int DV>
__global__ void __launch_bounds__(256)
attention_decode_maps_merge_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml,
                                   const bf16* __restrict__ q, int q_stride, bf16* __restrict__ out, int nsplit, int nh,
                                   int nkv, int G, DecodeMaps dm) {
  __shared__ float sm[DEC_MAXSPLIT][DEC_MAXG], sl[DEC_MAXSPLIT][DEC_MAXG], sf[DEC_MAXSPLIT][DEC_MAXG];
  __shared__ float sinv[DEC_MAXG];
  __shared__ float so[DEC_MAXG][DV];
  const int kvh = blockIdx.x, seq = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const size_t base = ((size_t)seq * nkv + kvh) * nsplit;
  for (int i = threadIdx.x; i < nsplit * G; i += blockDim.x) {
    const int sp = i / G, g = i - sp * G;
    sm[sp][g] = part_ml[((base + sp) * G + g) * 2];
    sl[sp][g] = part_ml[((base + sp) * G + g) * 2 + 1];
  }
  __syncthreads();
  if (threadIdx.x < G) {
    const int g = threadIdx.x;
    float M = -INFINITY;
    for (int sp = 0; sp < nsplit; ++sp) M = fmaxf(M, sm[sp][g]);
    float L = 0.f;
    for (int sp = 0; sp < nsplit; ++sp) {
      const float f = sm[sp][g] > -INFINITY ? __builtin_amdgcn_exp2f(sm[sp][g] - M) : 0.f;
      sf[sp][g] = f;
      L += sl[sp][g] * f;
    }
    sinv[g] = 1.0f / L;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < G * DV; i += blockDim.x) {
    const int g = i / DV, j = i - g * DV;
    float o = 0.f;
    for (int sp = 0; sp < nsplit; ++sp) o += part_o[((base + sp) * G + g) * DV + j] * sf[sp][g];
    so[g][j] = o * sinv[g];
  }
  __syncthreads();
  for (int hq = wave; hq < G / 2; hq += 4) {
    const int h = kvh * (G / 2) + hq;
    const float gate = dm.gate_col >= 0 ? 1.f / (1.f + expf(-to_f32(q[(size_t)seq * q_stride + dm.gate_col + h]))) : 1.f;
    finish_maps<DV>(so[2 * hq], so[2 * hq + 1], dm, gate, out + ((size_t)seq * (nh / 2) + h) * DV, lane);
  }
}

// Compute units of the device, asked for once.
inline int decode_compute_units() {
  static int cus = 0;
  if (cus == 0) {
    int dev = 0, n = 0;
    if (hipGetDevice(&dev) != hipSuccess || hipDeviceGetAttribute(&n, hipDeviceAttributeMultiprocessorCount, dev) != hipSuccess || n <= 0)
      n = 256;
    cus = n;
  }
  return cus;
}
