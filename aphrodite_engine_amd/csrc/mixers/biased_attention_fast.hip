// The plain bf16 forms (no mask beyond causality, no soft cap, no sink, per-head gate) and the host-side choices.
#include "biased_attention_fast.h"

namespace aphro {

bool dba_prefill_supported(int dim, int vdim) {
  auto ok = [](int d) { return d == 32 || d == 64 || d == 96 || d == 128; };
  return ok(dim) && ok(vdim);
}

bool dba_decode_supported(int heads, int kv_heads, int dim, int vdim) {
  return (dim & 7) == 0 && (vdim & 7) == 0 && decode_chl(dim, vdim) <= 5;
}

int dba_decode_units(int heads, int kv_heads, int dim, int vdim) {
  const int qh = decode_qh(heads, kv_heads, decode_chl(dim, vdim));
  return kv_heads * ((heads / kv_heads + qh - 1) / qh);
}

// Key splits of the decode kernel: enough workgroups to fill the chip, at least four 64-key tiles (one per wave) each.
int dba_decode_splits(int64_t num_tokens, int units, int max_kv_len, int64_t ws_floats, int heads, int vdim) {
  const int tiles = (max_kv_len + 63) / 64;
  int64_t n = (1024 + num_tokens * units - 1) / (num_tokens * units);
  if (n > tiles / 4) n = tiles / 4;
  if (n > 8) n = 8;
  while (n > 1 && num_tokens * heads * n * (2 + vdim) > ws_floats) --n;
  return n < 1 ? 1 : (int)n;
}

template void dba_prefill_launch<DBA_PLAIN>(const DBAParams&, int, int, hipStream_t);
template void dba_decode_launch<DBA_PLAIN>(const DBAParams&, int64_t, int, hipStream_t);

}  // namespace aphro
