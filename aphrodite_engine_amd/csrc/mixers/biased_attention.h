// Parameters and launchers of the distance-biased attention's bf16 fast paths (biased_attention_fast.h).
#pragma once
#include "mixers_common.h"

namespace aphro {

struct DBAParams {
  uint16_t* out;
  const uint16_t* q;
  const uint16_t* gate;
  const uint16_t* k_cache;
  const uint16_t* v_cache;
  const int32_t* block_tables;
  const int32_t* q_start;
  const int32_t* q_len;
  const int32_t* ctx_len;
  const int32_t* seq_of_token;
  const float* bias_lut;
  int64_t out_stride, q_stride, gate_stride, num_blocks;
  int max_blocks, block_size, heads, kv_heads, dim, vdim, lut_len, temp_every, min_len;
  float scale, temp_coef, out_scale;
  float* ws;          // decode split partials [T, heads, nsplit, 2 + vdim]
  int bs_shift;       // log2(block_size), or -1 when it is no power of two
  int max_tiles;      // prompt kernel: 64-row tiles of the longest segment
  // the forms with a mask, a soft cap, a sink or an elementwise gate
  int window, chunk;  // 0: none
  float softcap;      // 0: none
  float cap_in, cap_out;   // prompt kernel: cap tanh(x / cap) of scores in units of ln 2 = cap_out - 2 cap_out / (2^(x cap_in) + 1)
  const float* sink;  // fp32 [heads] or null
  int gate_cols;      // 1: gate [T, heads * vdim], 0: gate [T, heads]
  int vec4;           // out (and an elementwise gate) can be accessed 8 bytes at a time
};

bool dba_prefill_supported(int dim, int vdim);
bool dba_decode_supported(int heads, int kv_heads, int dim, int vdim);
// workgroups per decoded row (before the key range is split)
int dba_decode_units(int heads, int kv_heads, int dim, int vdim);
int dba_decode_splits(int64_t num_tokens, int units, int max_kv_len, int64_t ws_floats, int heads, int vdim);
// The forms of the kernels, a translation unit each: causal with a gate per head at most; window / chunk, soft cap, sink and elementwise
// gate, chosen at run time; causal with an elementwise gate.
enum DBAForm { DBA_PLAIN = 0, DBA_MASKED = 1, DBA_GATED = 2 };
template <int FORM>
void dba_prefill_launch(const DBAParams& p, int max_q_len, int num_seqs, hipStream_t st);
template <int FORM>
void dba_decode_launch(const DBAParams& p, int64_t num_tokens, int nsplit, hipStream_t st);
constexpr int DBA_MFMA_MIN_LEN = 8;     // segments at least this long go to the matrix-core kernel

}  // namespace aphro
