// Decode attention: one query token per sequence over its paged keys and values, bfloat16 cache.
//
// The step reads every cached key and value of the live sequences once; that stream is all the
// work there is, and for a few hundred keys the kernel's time is a chain of memory round trips
// (position, page number, rows), so the chain is kept short: a wavefront issues all the loads of a
// tile of 64 keys, keys and values, before it computes anything, and (where registers allow) the next
// tile's loads before it computes the current one.
//
// A block owns (split, key head, sequence): a contiguous share of the sequence's keys, for all G
// query heads that share the key head, so keys and values are read once per group.  Inside a block
// each wavefront takes tiles of 64 keys.  Scores run on the matrix cores (v_mfma_f32_16x16x32_bf16:
// 16 keys x 16 head columns, of which G are used, per instruction), with the key rows loaded straight
// in operand order and the queries held in registers.  Softmax runs online per head (running maximum
// and sum, base-2 exponentials of scores scaled by log2 e).  Values: lane = (key group, chunk of 8
// features); 16-byte loads of V rows, probabilities broadcast from LDS.  Wavefronts, then splits, are merged by the usual (max, sum, accumulator) rule
// in a fixed order.  With one split the block writes the output itself; with more, each block writes
// its partial (accumulator, max, sum) and a second small kernel merges them in split order.  (Merging
// in the last block to arrive would save that launch, but the device-wide fence it needs writes back
// and invalidates the L2 in every block, which costs far more than the launch.)  A block has eight
// wavefronts, so that for contexts of up to about a thousand keys one block per (sequence, key head)
// covers them in a pass or two and no merge kernel is needed.  Scores, maxima, sums and accumulators
// are float32.
//
// Everything that changes between steps (positions, block table) is read from device memory, so the
// launch can be recorded into a graph.  q (T, q_stride), head h at [h D, (h+1) D); caches
// (pages, nkv, page_size, D); out (T, nh D).  Window: keys lo..pos with lo = pos - window + 1.
#include "attention_decode_impl.h"
#include "no_alloc.h"
#include <mutex>

// Merge the splits of each (sequence, head), in split order.  One block per (sequence, key head).  The splits'
// maxima and sums go through LDS, so that each head's weights are computed once and the loads of the partial
// outputs are independent of one another.
__global__ void attention_decode_merge_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml,
                                              bf16* __restrict__ out, int nsplit, int nh, int nkv, int G, int D,
                                              int out_tiles, int sink, const float* __restrict__ sinks) {
  __shared__ float sm[DEC_MAXSPLIT][DEC_MAXG], sl[DEC_MAXSPLIT][DEC_MAXG], sf[DEC_MAXSPLIT][DEC_MAXG];
  __shared__ float sinv[DEC_MAXG];
  const int kvh = blockIdx.x, seq = blockIdx.y;
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
      const float f = sm[sp][g] > -INFINITY ? __builtin_amdgcn_exp2f(sm[sp][g] - M) : 0.f;   // maxima are in base-2 units
      sf[sp][g] = f;
      L += sl[sp][g] * f;
    }
    if (sink || sinks) L += M > -INFINITY ? __builtin_amdgcn_exp2f((sinks ? sinks[kvh * G + g] * DEC_LOG2E : 0.f) - M) : 1.f;
    sinv[g] = 1.0f / L;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < G * D; i += blockDim.x) {
    const int g = i / D, j = i - g * D;
    float o = 0.f;
    int sp = 0;
    for (; sp + 8 <= nsplit; sp += 8) {
      float v[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) v[u] = part_o[((base + sp + u) * G + g) * D + j];
#pragma unroll
      for (int u = 0; u < 8; ++u) o += v[u] * sf[sp + u][g];
    }
    for (; sp < nsplit; ++sp) o += part_o[((base + sp) * G + g) * D + j] * sf[sp][g];
    out[out_index(seq, (kvh * G + g) * D + j, nh * D, out_tiles)] = f32_to_bf16(o * sinv[g]);
  }
}

#define DEC_WAVES 8

// Wavefronts a block: eight, so that one block covers about a thousand keys in a pass or two; four where the grid
// holds more blocks than the chip has compute units (many sequences): blocks of four leave a lane's registers
// to two blocks a compute unit, whose chains of round trips then overlap (measured at 48 and at 64 sequences of
// 8 key heads: 18.5 against 23.8 us, 21 against 27).
template <int D, int RAW, int WV>
static int launch_decode_w(int G, dim3 grid, hipStream_t stream, const bf16* q, int q_stride, bf16* kc, bf16* vc,
                         const int* positions, const int* bt, int max_blocks, int page_size, unsigned page_magic,
                         int window, float scale, bf16* out, float* part_o, float* part_ml, int nh, int nkv,
                         int out_tiles, DecodeRaw raw) {
#define GS_RUN(GG)                                                                                                     \
  attention_decode_kernel<D, GG, WV, RAW><<<grid, WV * 64, 0, stream>>>(                                 \
      q, q_stride, kc, vc, positions, bt, max_blocks, page_size, page_magic, window, scale, out, part_o, part_ml, nh, \
      nkv, out_tiles, raw, DecodeMaps{})
  switch (G) {
    case 1: GS_RUN(1); break;
    case 2: GS_RUN(2); break;
    case 3: GS_RUN(3); break;
    case 4: GS_RUN(4); break;
    case 5: GS_RUN(5); break;
    case 6: GS_RUN(6); break;
    case 7: GS_RUN(7); break;
    case 8: GS_RUN(8); break;
    default: return -1;
  }
#undef GS_RUN
  return 0;
}

template <int D, int RAW>
static int launch_decode(int G, dim3 grid, hipStream_t stream, const bf16* q, int q_stride, bf16* kc, bf16* vc,
                         const int* positions, const int* bt, int max_blocks, int page_size, unsigned page_magic,
                         int window, float scale, bf16* out, float* part_o, float* part_ml, int nh, int nkv,
                         int out_tiles, DecodeRaw raw) {
  const long blocks = (long)grid.x * grid.y * grid.z;
  if (D <= 64 && blocks > 1L * decode_compute_units())
    return launch_decode_w<D, RAW, 4>(G, grid, stream, q, q_stride, kc, vc, positions, bt, max_blocks, page_size, page_magic,
                                      window, scale, out, part_o, part_ml, nh, nkv, out_tiles, raw);
  return launch_decode_w<D, RAW, DEC_WAVES>(G, grid, stream, q, q_stride, kc, vc, positions, bt, max_blocks, page_size,
                                            page_magic, window, scale, out, part_o, part_ml, nh, nkv, out_tiles, raw);
}

// Whether this kernel takes the sizes: head widths 16, 32, 64, 96, 128 and groups of up to 8 heads.
extern "C" int gs_attention_decode_supports(int nh, int nkv, int d) {
  if (nkv <= 0 || nh % nkv) return 0;
  int g = nh / nkv;
  return (d == 16 || d == 32 || d == 64 || d == 96 || d == 128) && g >= 1 && g <= DEC_MAXG;
}

// Floats of workspace for nseq sequences: partial outputs, then (max, sum) pairs.
extern "C" long gs_attention_decode_workspace(int nseq, int nh, int nkv, int d, int nsplit) {
  return (long)nseq * nh * nsplit * (d + 2);
}

static int decode_entry(const void* q, int q_stride, void* kcache, void* vcache, const int* positions,
                        const int* block_table, int max_blocks, int page_size, int window, float scale, void* out,
                        int out_tiled, float* workspace, int nseq, int nh, int nkv, int d, int nsplit,
                        const DecodeRaw* raw, hipStream_t stream, int chunk = 0, int sink = 0, float softcap = 0.f,
                        int keep_first = 0, const float* sinks = nullptr) {
  GS_REQUIRE(chunk >= 0, "attention_decode: bad chunk %d", chunk);
  GS_REQUIRE(softcap >= 0.f && keep_first >= 0 && !(sink && sinks), "attention_decode: bad cap, kept positions or sinks");
  GS_REQUIRE(keep_first == 0 || (window > 0 && chunk == 0), "attention_decode: kept first positions go with a window and no runs");
  GS_REQUIRE(!out_tiled || (nh * d) % 32 == 0, "attention_decode: tiled rows need a width that is a multiple of 32, not %d", nh * d);
  const int out_tiles = out_tiled ? gs_ceil_div(nseq, 16) : 0;
  GS_REQUIRE(gs_attention_decode_supports(nh, nkv, d), "attention_decode: sizes nh=%d nkv=%d d=%d are not taken", nh, nkv, d);
  GS_REQUIRE(nseq >= 0 && nseq <= 65535 && nkv <= 65535, "attention_decode: bad batch %d", nseq);
  GS_REQUIRE(nsplit >= 1 && nsplit <= 64, "attention_decode: %d splits outside [1, 64]", nsplit);
  GS_REQUIRE(page_size > 0 && max_blocks > 0 && window >= 0, "attention_decode: bad page_size/max_blocks/window");
  GS_REQUIRE(q_stride >= (raw ? nh + 2 * nkv : nh) * d, "attention_decode: q_stride %d below the row's width", q_stride);
  GS_REQUIRE(q_stride % 8 == 0 && ((uintptr_t)q & 15) == 0, "attention_decode: query rows must be 16-byte aligned");
  GS_REQUIRE((d * (int)sizeof(bf16)) % 16 == 0 && ((uintptr_t)kcache & 15) == 0 && ((uintptr_t)vcache & 15) == 0,
             "attention_decode: cache rows must be 16-byte aligned");
  if (nseq == 0) return 0;
  int G = nh / nkv;
  dim3 grid(nsplit, nkv, nseq);
  GS_REQUIRE(page_size >= 2 && (long)max_blocks * page_size * page_size < (1L << 32),
             "attention_decode: page_size %d with %d blocks a sequence is outside what the kernel's division takes", page_size, max_blocks);
  const unsigned page_magic = (unsigned)((1ull << 32) / (unsigned)page_size + 1);
  float* part_o = workspace;
  float* part_ml = workspace + (size_t)nseq * nh * nsplit * d;
  int rc = -1;
  DecodeRaw none = {};
  none.chunk = chunk;
  none.sink = sink ? 1 : 0;
  none.softcap = softcap;
  none.keep_first = keep_first;
  none.sinks = sinks;
  DecodeRaw with = raw ? *raw : none;
  with.chunk = chunk;
  with.sink = sink ? 1 : 0;
  with.softcap = softcap;
  with.keep_first = keep_first;
  with.sinks = sinks;
#define GS_ARGS                                                                                             \
  G, grid, stream, (const bf16*)q, q_stride, (bf16*)kcache, (bf16*)vcache, positions, block_table, max_blocks, \
      page_size, page_magic, window, scale, (bf16*)out, part_o, part_ml, nh, nkv, out_tiles
  if (raw) {
    switch (d) {
      case 64: rc = launch_decode<64, 1>(GS_ARGS, with); break;
      case 128: rc = launch_decode<128, 1>(GS_ARGS, with); break;
    }
  } else {
    switch (d) {
      case 16: rc = launch_decode<16, 0>(GS_ARGS, none); break;
      case 32: rc = launch_decode<32, 0>(GS_ARGS, none); break;
      case 64: rc = launch_decode<64, 0>(GS_ARGS, none); break;
      case 96: rc = launch_decode<96, 0>(GS_ARGS, none); break;
      case 128: rc = launch_decode<128, 0>(GS_ARGS, none); break;
    }
  }
#undef GS_ARGS
  GS_REQUIRE(rc == 0, "attention_decode: no kernel for group %d and head width %d", G, d);
  GS_LAUNCH_CHECK("attention_decode");
  if (nsplit > 1) {
    dim3 mgrid(nkv, nseq);
    attention_decode_merge_kernel<<<mgrid, 256, 0, stream>>>(part_o, part_ml, (bf16*)out, nsplit, nh, nkv, G, d, out_tiles,
                                                             sink ? 1 : 0, sinks);
    GS_LAUNCH_CHECK("attention_decode_merge");
  }
  return 0;
}

extern "C" int gs_attention_decode(const void* q, int q_stride, const void* kcache, const void* vcache,
                                   const int* positions, const int* block_table, int max_blocks, int page_size,
                                   int window, float scale, void* out, int out_tiled, float* workspace, int nseq, int nh,
                                   int nkv, int d, int nsplit, hipStream_t stream) {
  return decode_entry(q, q_stride, (void*)kcache, (void*)vcache, positions, block_table, max_blocks, page_size, window,
                      scale, out, out_tiled, workspace, nseq, nh, nkv, d, nsplit, nullptr, stream);
}

// The same with runs of positions and a sink (see DecodeRaw).
extern "C" int gs_attention_decode_runs(const void* q, int q_stride, const void* kcache, const void* vcache,
                                        const int* positions, const int* block_table, int max_blocks, int page_size,
                                        int window, float scale, void* out, int out_tiled, float* workspace, int nseq,
                                        int nh, int nkv, int d, int nsplit, int chunk, int sink, hipStream_t stream) {
  return decode_entry(q, q_stride, (void*)kcache, (void*)vcache, positions, block_table, max_blocks, page_size, window,
                      scale, out, out_tiled, workspace, nseq, nh, nkv, d, nsplit, nullptr, stream, chunk, sink);
}

// The same with a cap on the scores, kept first positions and sinks of the heads' own as well (see DecodeRaw).
extern "C" int gs_attention_decode_rules(const void* q, int q_stride, const void* kcache, const void* vcache,
                                         const int* positions, const int* block_table, int max_blocks, int page_size,
                                         int window, float scale, void* out, int out_tiled, float* workspace, int nseq,
                                         int nh, int nkv, int d, int nsplit, int chunk, int sink, float softcap,
                                         int keep_first, const float* sinks, hipStream_t stream) {
  return decode_entry(q, q_stride, (void*)kcache, (void*)vcache, positions, block_table, max_blocks, page_size, window,
                      scale, out, out_tiled, workspace, nseq, nh, nkv, d, nsplit, nullptr, stream, chunk, sink, softcap,
                      keep_first, sinks);
}

// ---- the entry point that allocates nothing (declared and described in no_alloc.h)
//
// `scratch` is the name of the device array as host code sees it: a stand-in, not a device address.  Its address on
// the current GPU comes from hipGetSymbolAddress, once per device with that device current (each GPU holds its own
// copy at its own address), and only that pointer goes to kernels.
static __device__ __align__(256) float scratch[GS_DECODE_STATIC_FLOATS];

#define GS_MAX_DEVICES 64
static float* g_scratch_ptr[GS_MAX_DEVICES];
static std::mutex g_scratch_mutex;

static int static_workspace(float** ptr) {
  int dev = -1;
  hipError_t e = hipGetDevice(&dev);
  GS_REQUIRE(e == hipSuccess, "attention_decode_static: no current device: %s", hipGetErrorString(e));
  GS_REQUIRE(dev >= 0 && dev < GS_MAX_DEVICES, "attention_decode_static: device %d outside [0, %d)", dev, GS_MAX_DEVICES);
  std::lock_guard<std::mutex> lock(g_scratch_mutex);
  if (g_scratch_ptr[dev] == nullptr) {
    float* p = nullptr;
    e = hipGetSymbolAddress((void**)&p, HIP_SYMBOL(scratch));
    GS_REQUIRE(e == hipSuccess && p != nullptr, "attention_decode_static: the static workspace has no address on device %d: %s",
               dev, hipGetErrorString(e));
    g_scratch_ptr[dev] = p;
  }
  *ptr = g_scratch_ptr[dev];
  return 0;
}

extern "C" int gs_attention_decode_static(const void* q, int q_stride, const void* kcache, const void* vcache,
                                          const int* positions, const int* block_table, int max_blocks, int page_size,
                                          int window, float scale, void* out, int out_tiled, int nseq, int nh, int nkv,
                                          int d, int nsplit, hipStream_t stream) {
  GS_REQUIRE(nseq >= 0 && nh > 0 && nkv > 0 && d > 0 && nsplit >= 1 && nsplit <= 64,
             "attention_decode_static: bad sizes nseq=%d nh=%d nkv=%d d=%d nsplit=%d", nseq, nh, nkv, d, nsplit);
  const long need = gs_attention_decode_workspace(nseq, nh, nkv, d, nsplit);
  GS_REQUIRE(need <= (long)GS_DECODE_STATIC_FLOATS,
             "attention_decode_static: %ld floats of workspace needed (nseq=%d nh=%d d=%d nsplit=%d), the static one holds %ld",
             need, nseq, nh, d, nsplit, (long)GS_DECODE_STATIC_FLOATS);
  float* ws = nullptr;
  if (static_workspace(&ws) != 0) return -1;
  return decode_entry(q, q_stride, (void*)kcache, (void*)vcache, positions, block_table, max_blocks, page_size, window,
                      scale, out, out_tiled, ws, nseq, nh, nkv, d, nsplit, nullptr, stream);
}

// Whether the kernel also takes the head norms, the rotation and the cache write: heads of 64 or 128 rotated whole.
extern "C" int gs_attention_decode_raw_supports(int nh, int nkv, int d, int rotary_dim) {
  return gs_attention_decode_supports(nh, nkv, d) && (d == 64 || d == 128) && rotary_dim == d;
}

// qkv (nseq, q_stride): the rows of q|k|v as their product left them.  The kernel norms and rotates q and the new
// key, writes the new key and value into their pages (unless write_kv is 0), and attends.
extern "C" int gs_attention_decode_raw(const void* qkv, int q_stride, void* kcache, void* vcache, const int* positions,
                                       const int* block_table, int max_blocks, int page_size, int window, float scale,
                                       const float* qw, const float* kw, float eps, const float* cos_t,
                                       const float* sin_t, int rotary_dim, int write_kv, void* out, int out_tiled,
                                       float* workspace, int nseq, int nh, int nkv, int d, int nsplit,
                                       hipStream_t stream) {
  GS_REQUIRE(gs_attention_decode_raw_supports(nh, nkv, d, rotary_dim), "attention_decode_raw: sizes nh=%d nkv=%d d=%d rotary=%d are not taken", nh, nkv, d, rotary_dim);
  GS_REQUIRE((qw == nullptr) == (kw == nullptr) && cos_t && sin_t, "attention_decode_raw: q and k norm weights come together; the rotation needs its tables");
  GS_REQUIRE((((uintptr_t)qw | (uintptr_t)kw | (uintptr_t)cos_t | (uintptr_t)sin_t) & 15) == 0, "attention_decode_raw: weights and tables must be 16-byte aligned");
  DecodeRaw raw = {qw, kw, eps, cos_t, sin_t, write_kv};
  return decode_entry(qkv, q_stride, kcache, vcache, positions, block_table, max_blocks, page_size, window, scale, out,
                      out_tiled, workspace, nseq, nh, nkv, d, nsplit, &raw, stream);
}
