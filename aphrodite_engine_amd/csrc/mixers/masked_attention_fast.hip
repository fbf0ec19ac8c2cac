// The bf16 forms under a sliding window or chunks, with a soft cap, a sink or an elementwise gate.
#include "biased_attention_fast.h"

namespace aphro {

template void dba_prefill_launch<DBA_MASKED>(const DBAParams&, int, int, hipStream_t);
template void dba_decode_launch<DBA_MASKED>(const DBAParams&, int64_t, int, hipStream_t);

}  // namespace aphro
