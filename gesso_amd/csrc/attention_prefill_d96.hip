// Prompt attention for heads 96 wide.
#include "attention_prefill_impl.h"

int gs_attention_prefill_d96(const PrefillCall& c) { return prefill_for_width<96>(c); }
