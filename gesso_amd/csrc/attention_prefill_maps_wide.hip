// Prompt attention over two maps, values 128 wide.
#include "attention_prefill_impl.h"

int gs_attention_prefill_maps_wide(const PrefillCall& c, const MapsEnd& me, int d, int dv) {
  if (d == 32 && dv == 128) return prefill_maps_for_width<32, 128>(c, me);
  if (d == 64 && dv == 128) return prefill_maps_for_width<64, 128>(c, me);
  if (d == 128 && dv == 128) return prefill_maps_for_width<128, 128>(c, me);
  return -1;
}
