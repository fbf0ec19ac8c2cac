// The causal bf16 forms with an elementwise gate: no mask beyond causality, no soft cap, no sink.
#include "biased_attention_fast.h"

namespace aphro {

template void dba_prefill_launch<DBA_GATED>(const DBAParams&, int, int, hipStream_t);
template void dba_decode_launch<DBA_GATED>(const DBAParams&, int64_t, int, hipStream_t);

}  // namespace aphro
