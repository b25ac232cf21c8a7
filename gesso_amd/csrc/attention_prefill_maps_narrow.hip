// Prompt attention over two maps, values up to 64 wide.
#include "attention_prefill_impl.h"

int gs_attention_prefill_maps_narrow(const PrefillCall& c, const MapsEnd& me, int d, int dv) {
  if (d == 32 && dv == 32) return prefill_maps_for_width<32, 32>(c, me);
  if (d == 32 && dv == 64) return prefill_maps_for_width<32, 64>(c, me);
  if (d == 64 && dv == 64) return prefill_maps_for_width<64, 64>(c, me);
  return -1;
}
