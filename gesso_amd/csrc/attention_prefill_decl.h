// What the entry point of the prompt attention hands to the kernels of one head width.
#pragma once
#include "common.h"

struct PrefillCall {
  const bf16 *q, *kc, *vc;
  const int *positions, *tile_seq, *tile_row, *tile_n, *bt;
  int q_stride, max_blocks, page_size, window, nh, nkv, tile_rows, ntiles;
  int chunk, sink, keep_first;
  unsigned page_magic;
  float scale, softcap;
  const float* sinks;
  bf16* out;
  hipStream_t stream;
};

// What the end of attention over two maps needs: the second map's share, the norm's eps, what the normed difference is
// multiplied by, where in the query's row the heads' gates stand (< 0: none), and into how many blocks a key head's group
// of query heads is cut.
struct MapsEnd {
  float lam, eps, out_scale;
  int gate_col, parts;
};

int gs_attention_prefill_d32(const PrefillCall& c);
int gs_attention_prefill_d64(const PrefillCall& c);
int gs_attention_prefill_d96(const PrefillCall& c);
int gs_attention_prefill_d128(const PrefillCall& c);
int gs_attention_prefill_maps_narrow(const PrefillCall& c, const MapsEnd& me, int d, int dv);
int gs_attention_prefill_maps_wide(const PrefillCall& c, const MapsEnd& me, int d, int dv);
