// Prompt attention on the matrix cores: the entry point; the kernels are in attention_prefill_impl.h, compiled
// per head width in attention_prefill_d*.hip.
#include "attention_prefill_decl.h"


// Head widths 32, 64, 96, 128; groups of 1 to 8 heads (the block has one wavefront per head of the group).
extern "C" int gs_attention_prefill_supports(int nh, int nkv, int d) {
  if (nkv <= 0 || nh % nkv) return 0;
  int g = nh / nkv;
  return (d == 32 || d == 64 || d == 96 || d == 128) && g >= 1 && g <= 8;
}

extern "C" int gs_attention_prefill(const void* q, int q_stride, const void* kcache, const void* vcache,
                                    const int* positions, const int* tile_seq, const int* tile_row,
                                    const int* tile_n, int ntiles, const int* block_table, int max_blocks,
                                    int page_size, int window, float scale, void* out, int nh, int nkv, int d,
                                    int tile_rows, int chunk, int sink, float softcap, int keep_first,
                                    const float* sinks, hipStream_t stream) {
  GS_REQUIRE(chunk >= 0, "attention_prefill: bad chunk %d", chunk);
  GS_REQUIRE(softcap >= 0.f && keep_first >= 0 && !(sink && sinks), "attention_prefill: bad cap, kept positions or sinks");
  GS_REQUIRE(keep_first == 0 || (window > 0 && chunk == 0), "attention_prefill: kept first positions go with a window and no runs");
  GS_REQUIRE(gs_attention_prefill_supports(nh, nkv, d), "attention_prefill: sizes nh=%d nkv=%d d=%d are not taken", nh, nkv, d);
  GS_REQUIRE(ntiles >= 0 && nkv > 0 && (long)ntiles * nkv < (1L << 31), "attention_prefill: %d tiles x %d key heads are too many blocks", ntiles, nkv);
  GS_REQUIRE(tile_rows == 16 || tile_rows == 32, "attention_prefill: tiles hold 16 or 32 queries, not %d", tile_rows);
  GS_REQUIRE(page_size > 0 && max_blocks > 0 && window >= 0, "attention_prefill: bad page_size/max_blocks/window");
  GS_REQUIRE(q_stride >= nh * d && q_stride % 8 == 0 && ((uintptr_t)q & 15) == 0, "attention_prefill: q rows must be 16-byte aligned");
  GS_REQUIRE(((uintptr_t)kcache & 15) == 0 && ((uintptr_t)vcache & 15) == 0 && ((uintptr_t)out & 7) == 0,
             "attention_prefill: cache and output must be aligned");
  // the kernel divides by page_size with one multiplication, exact while key index x page_size < 2^32
  GS_REQUIRE(page_size >= 2 && (long)max_blocks * page_size * page_size < (1L << 32),
             "attention_prefill: page_size %d with %d blocks a sequence is outside what the kernel's division takes", page_size, max_blocks);
  if (ntiles == 0) return 0;
  const unsigned page_magic = (unsigned)((1ull << 32) / (unsigned)page_size + 1);
  PrefillCall c = {(const bf16*)q, (const bf16*)kcache, (const bf16*)vcache, positions, tile_seq, tile_row, tile_n,
                   block_table, q_stride, max_blocks, page_size, window, nh, nkv, tile_rows, ntiles, chunk, sink ? 1 : 0,
                   keep_first, page_magic, scale, softcap, sinks, (bf16*)out, stream};
  int rc = -1;
  switch (d) {
    case 32: rc = gs_attention_prefill_d32(c); break;
    case 64: rc = gs_attention_prefill_d64(c); break;
    case 96: rc = gs_attention_prefill_d96(c); break;
    case 128: rc = gs_attention_prefill_d128(c); break;
  }
  GS_REQUIRE(rc == 0, "attention_prefill: no kernel for this group size");
  GS_LAUNCH_CHECK("attention_prefill");
  return 0;
}

// How many query heads of a key head's group a block of the two-map kernels takes (1, 2 or 4), for a group of `rep` heads.
static int maps_heads_a_block(int rep) { return rep % 4 == 0 ? 4 : (rep % 2 == 0 ? 2 : 1); }

// The kernels for two maps a head: maps 32, 64 or 128 features wide, values 32, 64 or 128 (not every pair of them).
extern "C" int gs_attention_prefill_maps_supports(int nh, int nkv, int d, int dv) {
  if (nkv <= 0 || nh % nkv) return 0;
  return (dv == 128 && (d == 32 || d == 64 || d == 128)) || (dv == 64 && (d == 32 || d == 64)) || (dv == 32 && d == 32);
}

// Attention over two maps for prompt portions (see attention_maps.hip for the operands and the definition); nh query heads,
// maps of d features, values of dv.
extern "C" int gs_attention_prefill_maps(const void* q, int q_stride, const void* kcache, const void* vcache,
                                         const int* positions, const int* tile_seq, const int* tile_row,
                                         const int* tile_n, int ntiles, const int* block_table, int max_blocks,
                                         int page_size, int window, float scale, float lam, float eps, float out_scale,
                                         int gate_col, void* out, int nh, int nkv, int d, int dv, int tile_rows,
                                         hipStream_t stream) {
  GS_REQUIRE(gs_attention_prefill_maps_supports(nh, nkv, d, dv), "attention_prefill_maps: sizes nh=%d nkv=%d d=%d dv=%d are not taken", nh, nkv, d, dv);
  const int per = maps_heads_a_block(nh / nkv), parts = nh / nkv / per;
  GS_REQUIRE(ntiles >= 0 && (long)ntiles * nkv * parts < (1L << 31), "attention_prefill_maps: %d tiles x %d are too many blocks", ntiles, nkv * parts);
  GS_REQUIRE(tile_rows == 16 || tile_rows == 32, "attention_prefill_maps: tiles hold 16 or 32 queries, not %d", tile_rows);
  GS_REQUIRE(page_size > 0 && max_blocks > 0 && window >= 0, "attention_prefill_maps: bad page_size/max_blocks/window");
  GS_REQUIRE(eps > 0.f, "attention_prefill_maps: eps must be positive");
  GS_REQUIRE(q_stride >= 2 * nh * d && q_stride % 8 == 0 && ((uintptr_t)q & 15) == 0, "attention_prefill_maps: q rows must be 16-byte aligned");
  GS_REQUIRE(gate_col < 0 || gate_col + nh <= q_stride, "attention_prefill_maps: the gates lie outside the rows of %d", q_stride);
  GS_REQUIRE(((uintptr_t)kcache & 15) == 0 && ((uintptr_t)vcache & 15) == 0 && ((uintptr_t)out & 7) == 0,
             "attention_prefill_maps: cache and output must be aligned");
  GS_REQUIRE(page_size >= 2 && (long)max_blocks * page_size * page_size < (1L << 32),
             "attention_prefill_maps: page_size %d with %d blocks a sequence is outside what the kernel's division takes", page_size, max_blocks);
  if (ntiles == 0) return 0;
  const unsigned page_magic = (unsigned)((1ull << 32) / (unsigned)page_size + 1);
  PrefillCall c = {(const bf16*)q, (const bf16*)kcache, (const bf16*)vcache, positions, tile_seq, tile_row, tile_n,
                   block_table, q_stride, max_blocks, page_size, window, 2 * nh, nkv * parts, tile_rows, ntiles, 0, 0,
                   0, page_magic, scale, 0.f, nullptr, (bf16*)out, stream};
  const MapsEnd me = {lam, eps, out_scale, gate_col, parts};
  const int rc = dv == 128 ? gs_attention_prefill_maps_wide(c, me, d, dv) : gs_attention_prefill_maps_narrow(c, me, d, dv);
  GS_REQUIRE(rc == 0, "attention_prefill_maps: no kernel for these sizes");
  GS_LAUNCH_CHECK("attention_prefill_maps");
  return 0;
}
