// Decode attention over two maps a head: the launches (the kernels are in attention_decode_impl.h; attention_maps.hip has
// the operands and the definition).
#include "attention_decode_impl.h"

struct MapsDecodeCall {
  const bf16 *q, *kc, *vc;
  const int *positions, *bt;
  int q_stride, max_blocks, page_size, window, nseq, nh, nkv, nsplit;   // nh: maps of all heads; nkv: blocks a sequence
  unsigned page_magic;
  float scale;
  bf16* out;
  float *part_o, *part_ml;
  hipStream_t stream;
};

template <int D, int DV, int G, int W>
static void maps_launch(const MapsDecodeCall& c, const DecodeMaps& dm) {
  dim3 grid(c.nsplit, c.nkv, c.nseq);
  attention_decode_kernel<D, G, W, 0, DV, 2><<<grid, W * 64, 0, c.stream>>>(
      c.q, c.q_stride, (bf16*)c.kc, (bf16*)c.vc, c.positions, c.bt, c.max_blocks, c.page_size, c.page_magic, c.window,
      c.scale, c.out, c.part_o, c.part_ml, c.nh, c.nkv, 0, DecodeRaw{}, dm);
}

// Wavefronts a block: eight; four where the grid holds more blocks than the chip has compute units and rows are short
// enough for two blocks a unit (as for one map a head), and where the registers of eight do not hold two maps' rows.
template <int D, int DV>
static int maps_for_width(const MapsDecodeCall& c, const DecodeMaps& dm) {
  const int G = c.nh / c.nkv;
  const bool many = (long)c.nsplit * c.nkv * c.nseq > decode_compute_units();
  constexpr int EIGHT = D > 128 ? 4 : 8;
  const bool four = D > 128 || (D <= 64 && DV <= 64 && many);
#define GS_RUN(GG)                                    \
  do {                                                \
    if (four) maps_launch<D, DV, GG, 4>(c, dm);       \
    else maps_launch<D, DV, GG, EIGHT>(c, dm);          \
  } while (0)
  switch (G) {
    case 2: GS_RUN(2); break;
    case 4: GS_RUN(4); break;
    case 8: GS_RUN(8); break;
    default: return -1;
  }
#undef GS_RUN
  if (c.nsplit > 1)
    attention_decode_maps_merge_kernel<DV><<<dim3(c.nkv, c.nseq), 256, 0, c.stream>>>(c.part_o, c.part_ml, c.q, c.q_stride,
                                                                                      c.out, c.nsplit, c.nh, c.nkv, G, dm);
  return 0;
}

static int maps_heads_a_block(int rep) { return rep % 4 == 0 ? 4 : (rep % 2 == 0 ? 2 : 1); }

// Maps 16, 32, 64 or 128 features wide, values 32, 64 or 128 (not every pair of them).
extern "C" int gs_attention_decode_maps_supports(int nh, int nkv, int d, int dv) {
  if (nkv <= 0 || nh % nkv) return 0;
  return (dv == 128 && (d == 32 || d == 64 || d == 128)) || (dv == 64 && (d == 16 || d == 32 || d == 64)) ||
         (dv == 32 && (d == 16 || d == 32));
}

// How many blocks a sequence makes for one split of its keys (key heads times the parts their groups are cut into).
extern "C" int gs_attention_decode_maps_blocks(int nh, int nkv) {
  return nkv > 0 && nh % nkv == 0 ? nkv * (nh / nkv / maps_heads_a_block(nh / nkv)) : 0;
}

// Floats of workspace for nseq sequences: partial outputs of both maps, then (max, sum) pairs.
extern "C" long gs_attention_decode_maps_workspace(int nseq, int nh, int dv, int nsplit) {
  return (long)nseq * 2 * nh * nsplit * (dv + 2);
}

extern "C" int gs_attention_decode_maps(const void* q, int q_stride, const void* kcache, const void* vcache,
                                        const int* positions, const int* block_table, int max_blocks, int page_size,
                                        int window, float scale, float lam, float eps, float out_scale, int gate_col,
                                        void* out, float* workspace, int nseq, int nh, int nkv, int d, int dv, int nsplit,
                                        hipStream_t stream) {
  GS_REQUIRE(gs_attention_decode_maps_supports(nh, nkv, d, dv), "attention_decode_maps: sizes nh=%d nkv=%d d=%d dv=%d are not taken", nh, nkv, d, dv);
  const int per = maps_heads_a_block(nh / nkv), parts = nh / nkv / per;
  GS_REQUIRE(nseq >= 0 && nseq <= 65535 && nkv * parts <= 65535, "attention_decode_maps: bad batch %d", nseq);
  GS_REQUIRE(nsplit >= 1 && nsplit <= DEC_MAXSPLIT && (nsplit == 1 || workspace), "attention_decode_maps: %d splits outside [1, %d]", nsplit, DEC_MAXSPLIT);
  GS_REQUIRE(page_size > 0 && max_blocks > 0 && window >= 0, "attention_decode_maps: bad page_size/max_blocks/window");
  GS_REQUIRE(eps > 0.f, "attention_decode_maps: eps must be positive");
  GS_REQUIRE(q_stride >= 2 * nh * d && q_stride % 8 == 0 && ((uintptr_t)q & 15) == 0, "attention_decode_maps: query rows must be 16-byte aligned");
  GS_REQUIRE(gate_col < 0 || gate_col + nh <= q_stride, "attention_decode_maps: the gates lie outside the rows of %d", q_stride);
  GS_REQUIRE(((uintptr_t)kcache & 15) == 0 && ((uintptr_t)vcache & 15) == 0, "attention_decode_maps: cache rows must be 16-byte aligned");
  GS_REQUIRE(page_size >= 2 && (long)max_blocks * page_size * page_size < (1L << 32),
             "attention_decode_maps: page_size %d with %d blocks a sequence is outside what the kernel's division takes", page_size, max_blocks);
  if (nseq == 0) return 0;
  MapsDecodeCall c = {(const bf16*)q, (const bf16*)kcache, (const bf16*)vcache, positions, block_table, q_stride, max_blocks,
                      page_size, window, nseq, 2 * nh, nkv * parts, nsplit,
                      (unsigned)((1ull << 32) / (unsigned)page_size + 1), scale, (bf16*)out, workspace,
                      workspace ? workspace + (size_t)nseq * 2 * nh * nsplit * dv : nullptr, stream};
  const DecodeMaps dm = {lam, eps, out_scale, gate_col, parts};
  int rc = -1;
  if (dv == 32) rc = d == 16 ? maps_for_width<32, 32>(c, dm) : maps_for_width<64, 32>(c, dm);
  else if (dv == 64) rc = d == 16 ? maps_for_width<32, 64>(c, dm) : (d == 32 ? maps_for_width<64, 64>(c, dm) : maps_for_width<128, 64>(c, dm));
  else rc = d == 32 ? maps_for_width<64, 128>(c, dm) : (d == 64 ? maps_for_width<128, 128>(c, dm) : maps_for_width<256, 128>(c, dm));
  GS_REQUIRE(rc == 0, "attention_decode_maps: no kernel for these sizes");
  GS_LAUNCH_CHECK("attention_decode_maps");
  return 0;
}
