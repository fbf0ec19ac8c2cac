// What happens between the input product [q | k | v] of a rotary attention with short convolutions and its paged cache, in one launch:
//   every channel of q, k and v passes a short causal convolution over time (taps w[c, :], zeros before the sequence's start, the
//   inputs that precede a segment from the request's state slot);
//   optionally every query and key head is divided by its root mean square, times a weight per number shared by the heads;
//   the first rot_dims numbers of every query and key head turn by position * inv_freq[i], number i with number i + rot_dims / 2,
//   cos and sin times mscale; the rest of the head passes;
//   queries go to a dense output, keys and values into the token-major paged caches at the rows' slots;
//   the state slots take the last taps - 1 inputs of their sequences: in this launch when every segment is a single token (a slot's
//   channel then belongs to one thread, which has read it), in a second one otherwise.
// All fp32 from the projection's numbers to the one rounding at the store.
//
// A thread owns 8 neighbouring channels of one head and TOK consecutive rows (TOK + TAPS - 1 input rows and its taps are read once, 16
// bytes at a time); tph threads -- a power of two, within one wave -- share a head.  The angles of the workgroup's rows are worked out
// once, in LDS, for all its heads; rotation partners meet in LDS too, so that half the rotated part may be any number.
#include "mixers_common.h"

extern "C" int aphro_short_conv_state(void* state, const void* u, int64_t u_stride, const int32_t* state_slots, const int32_t* q_start,
                                      const int32_t* q_len, const int32_t* ctx_len, int num_seqs, int channels, int taps, int dtype,
                                      void* stream);

namespace aphro {

template <typename T>
struct ConvRotaryParams {
  typename T::storage* q_out;
  typename T::storage* k_cache;
  typename T::storage* v_cache;
  typename T::storage* state;
  const typename T::storage* u;
  const typename T::storage* w;
  const typename T::storage* q_weight;     // NULL (both): no norm
  const typename T::storage* k_weight;
  const int64_t* slot_mapping;
  const int32_t* state_slots;
  const int32_t* q_start;
  const int32_t* ctx_len;
  const int32_t* seq_of_token;
  const float* inv_freq;
  int64_t q_out_stride, u_stride, num_cache_rows, num_tokens;
  int heads, kv_heads, dim, vdim, rot_dims, tph, write_state;
  float mscale, eps;
};

template <typename T>
__device__ __forceinline__ void cr_load8(const typename T::storage* p, float* o) {
  if constexpr (sizeof(typename T::storage) == 2) {
    const u16x8 v = *reinterpret_cast<const u16x8*>(p);
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = T::to_f32(v[j]);
  } else {
    const f32x4 a = *reinterpret_cast<const f32x4*>(p), b = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      o[j] = a[j];
      o[4 + j] = b[j];
    }
  }
}
template <typename T>
__device__ __forceinline__ void cr_store8(typename T::storage* p, const float* v) {
  if constexpr (sizeof(typename T::storage) == 2) {
    *reinterpret_cast<u32x4*>(p) = u32x4{pack2_16<true>(v[0], v[1]), pack2_16<true>(v[2], v[3]), pack2_16<true>(v[4], v[5]), pack2_16<true>(v[6], v[7])};
  } else {
    *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
    *reinterpret_cast<f32x4*>(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
  }
}

// 8 numbers as they lie in memory (16 bytes of bf16, 32 of fp32): rows in flight take no more registers than that
template <typename T>
struct CRChunk {
  u32x4 v[sizeof(typename T::storage) / 2];
  __device__ __forceinline__ void load(const typename T::storage* p) {
#pragma unroll
    for (int i = 0; i < (int)(sizeof(typename T::storage) / 2); ++i) v[i] = reinterpret_cast<const u32x4*>(p)[i];
  }
  __device__ __forceinline__ void clear() {
#pragma unroll
    for (int i = 0; i < (int)(sizeof(typename T::storage) / 2); ++i) v[i] = u32x4{0, 0, 0, 0};
  }
  __device__ __forceinline__ void store(typename T::storage* p) const {
#pragma unroll
    for (int i = 0; i < (int)(sizeof(typename T::storage) / 2); ++i) reinterpret_cast<u32x4*>(p)[i] = v[i];
  }
  __device__ __forceinline__ void floats(float* o) const {
    if constexpr (sizeof(typename T::storage) == 2) {
      const u16x8 x = __builtin_bit_cast(u16x8, v[0]);
#pragma unroll
      for (int j = 0; j < 8; ++j) o[j] = T::to_f32(x[j]);
    } else {
      const f32x4 a = __builtin_bit_cast(f32x4, v[0]), b = __builtin_bit_cast(f32x4, v[1]);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        o[j] = a[j];
        o[4 + j] = b[j];
      }
    }
  }
};

constexpr int CR_THREADS = 256, CR_MAX_DIM = 512;

// LDS written by lanes of a wave and read by others of the same wave
__device__ __forceinline__ void cr_wave_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

template <typename T, int TAPS, int TOK>
__global__ __launch_bounds__(CR_THREADS) void conv_rotary_qk_norm_kv_write_kernel(ConvRotaryParams<T> p) {
  typedef typename T::storage S;
  extern __shared__ __attribute__((aligned(16))) float cr_lds[];
  float* xch = cr_lds;                                       // 8 numbers of every thread
  f32x2* turn = reinterpret_cast<f32x2*>(cr_lds + 8 * CR_THREADS);      // (cos, sin) of [row of the tile][pair]
  const int64_t t0 = (int64_t)blockIdx.x * TOK;
  const int half = p.rot_dims >> 1;
  // what the rows of the tile are (uniform over the workgroup), asked for together
  int seq[TOK], back0[TOK], ctx[TOK], sslot[TOK];
  int64_t cslot[TOK];
#pragma unroll
  for (int k = 0; k < TOK; ++k) {
    const int64_t t = t0 + k < p.num_tokens ? t0 + k : p.num_tokens - 1;
    seq[k] = p.seq_of_token[t];
    cslot[k] = p.slot_mapping[t];
  }
#pragma unroll
  for (int k = 0; k < TOK; ++k) {
    const int64_t t = t0 + k < p.num_tokens ? t0 + k : p.num_tokens - 1;
    back0[k] = (int)t - p.q_start[seq[k]];                   // rows of the segment ahead of this one
    ctx[k] = p.ctx_len[seq[k]];
    sslot[k] = TAPS > 1 ? p.state_slots[seq[k]] : 0;
  }
  for (int i = threadIdx.x; i < TOK * half; i += CR_THREADS) {
    const int64_t t = t0 + i / half;
    if (t >= p.num_tokens) break;
    const int s = p.seq_of_token[t];
    float c, sn;
    sincosf((float)(p.ctx_len[s] + (int)(t - p.q_start[s])) * p.inv_freq[i % half], &sn, &c);
    turn[i] = f32x2{c * p.mscale, sn * p.mscale};
  }
  __syncthreads();
  const int tph = p.tph, H = p.heads, G = p.kv_heads;
  const int unit = blockIdx.y * (CR_THREADS / tph) + threadIdx.x / tph, i0 = 8 * (threadIdx.x % tph);
  if (unit >= H + 2 * G) return;                             // whole groups of tph lanes leave together
  const bool is_q = unit < H, is_v = unit >= H + G;
  const int hd = is_q ? unit : (is_v ? unit - H - G : unit - H), n = is_v ? p.vdim : p.dim;
  const int C = (H + G) * p.dim + G * p.vdim;
  const int c0 = (is_v ? (H + G) * p.dim + hd * p.vdim : unit * p.dim) + i0;       // first channel (meaningful if work)
  const bool work = i0 < n;
  float wv[TAPS][8], nw[8];
  CRChunk<T> rows[TOK + TAPS - 1];
#pragma unroll
  for (int i = 0; i < 8; ++i) nw[i] = 1.f;
#pragma unroll
  for (int j = 0; j < TAPS; ++j)
#pragma unroll
    for (int i = 0; i < 8; ++i) wv[j][i] = 0.f;
  if (work) {
    float flat[8 * TAPS];
#pragma unroll
    for (int x = 0; x < TAPS; ++x) cr_load8<T>(p.w + (int64_t)c0 * TAPS + 8 * x, flat + 8 * x);
#pragma unroll
    for (int i = 0; i < 8; ++i)
#pragma unroll
      for (int j = 0; j < TAPS; ++j) wv[j][i] = flat[i * TAPS + j];
    if (!is_v && p.q_weight) cr_load8<T>((is_q ? p.q_weight : p.k_weight) + i0, nw);
  }
#pragma unroll
  for (int x = 0; x < TOK + TAPS - 1; ++x) {
    const int64_t gr = t0 - (TAPS - 1) + x;
    if (work && gr >= 0 && gr < p.num_tokens) rows[x].load(p.u + gr * p.u_stride + c0);
    else rows[x].clear();
  }
#pragma unroll
  for (int k = 0; k < TOK; ++k) {
    const int64_t t = t0 + k;
    if (t >= p.num_tokens) break;
    S* st = TAPS > 1 && work ? p.state + (int64_t)sslot[k] * (TAPS - 1) * C + c0 : nullptr;
    float acc[8];
    CRChunk<T> win[TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
      const int back = back0[k] - TAPS + 1 + j;              // row of the segment, negative: before it
      win[j] = rows[k + j];
      if (back < 0) {
        if (work && ctx[k] + back >= 0) win[j].load(st + (int64_t)(TAPS - 1 + back) * C);
        else win[j].clear();
      }
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[i] = 0.f;
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
      float x[8];
      win[j].floats(x);
#pragma unroll
      for (int i = 0; i < 8; ++i) acc[i] += wv[j][i] * x[i];
    }
    if (p.write_state && work) {
#pragma unroll
      for (int m = 0; m < TAPS - 1; ++m) win[m + 1].store(st + (int64_t)m * C);
    }
    const int64_t slot = cslot[k];
    const bool cached = slot >= 0 && slot < p.num_cache_rows;
    if (is_v) {
      if (work && cached) cr_store8<T>(p.v_cache + (slot * G + hd) * (int64_t)p.vdim + i0, acc);
      continue;
    }
    if (p.q_weight) {
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) ss += acc[i] * acc[i];     // lanes past the head hold zeros
      for (int o = tph >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
      const float f = 1.0f / sqrtf(ss / (float)p.dim + p.eps);
#pragma unroll
      for (int i = 0; i < 8; ++i) acc[i] *= f * nw[i];
    }
    if (half > 0) {
      float* mine = xch + 8 * threadIdx.x;
      const float* head = xch + 8 * (threadIdx.x - threadIdx.x % tph);
      *reinterpret_cast<f32x4*>(mine) = f32x4{acc[0], acc[1], acc[2], acc[3]};
      *reinterpret_cast<f32x4*>(mine + 4) = f32x4{acc[4], acc[5], acc[6], acc[7]};
      cr_wave_fence();
      if (i0 < 2 * half) {
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const int x = i0 + i;
          if (x < 2 * half) {
            const bool first = x < half;
            const f32x2 a = turn[k * half + (first ? x : x - half)];
            const float other = head[first ? x + half : x - half];
            acc[i] = first ? acc[i] * a[0] - other * a[1] : acc[i] * a[0] + other * a[1];
          }
        }
      }
      cr_wave_fence();                                       // everyone has read before the next row is laid down
    }
    if (!work) continue;
    if (is_q) cr_store8<T>(p.q_out + t * p.q_out_stride + (int64_t)hd * p.dim + i0, acc);
    else if (cached) cr_store8<T>(p.k_cache + (slot * G + hd) * (int64_t)p.dim + i0, acc);
  }
}

}  // namespace aphro

using namespace aphro;

extern "C" int aphro_conv_rotary_supported(int dim, int vdim, int taps) {
  return dim > 0 && dim % 8 == 0 && dim <= CR_MAX_DIM && vdim > 0 && vdim % 8 == 0 && vdim <= CR_MAX_DIM && taps >= 1 && taps <= 4;
}

extern "C" int aphro_conv_rotary_qk_norm_kv_write(void* q_out, int64_t q_out_stride, void* k_cache, void* v_cache, const int64_t* slot_mapping,
                                                  int64_t num_cache_rows, const void* u, int64_t u_stride, const void* w, void* state,
                                                  const int32_t* state_slots, const int32_t* q_start, const int32_t* q_len,
                                                  const int32_t* ctx_len, const int32_t* seq_of_token, const float* inv_freq, float mscale,
                                                  const void* q_weight, const void* k_weight, float eps, int64_t num_tokens, int num_seqs,
                                                  int max_q_len, int heads, int kv_heads, int dim, int vdim, int rot_dims, int taps, int dtype,
                                                  void* stream) {
  if (num_tokens == 0) return APHRO_OK;
  APHRO_CHECK(q_out && k_cache && v_cache && slot_mapping && u && w && q_start && q_len && ctx_len && seq_of_token && (rot_dims == 0 || inv_freq) &&
                  (q_weight == nullptr) == (k_weight == nullptr), "conv_rotary_qk_norm_kv_write: null argument");
  APHRO_CHECK(aphro_conv_rotary_supported(dim, vdim, taps), "conv_rotary_qk_norm_kv_write: heads of %d / %d (multiples of 8, <= %d), %d taps (1 .. 4)",
              dim, vdim, CR_MAX_DIM, taps);
  APHRO_CHECK(taps == 1 || (state && state_slots), "conv_rotary_qk_norm_kv_write: more than one tap needs the state slots");
  APHRO_CHECK(heads > 0 && kv_heads > 0 && rot_dims >= 0 && rot_dims <= dim && rot_dims % 2 == 0 && num_seqs > 0 && max_q_len > 0 &&
                  num_cache_rows > 0 && num_tokens <= 0x7fffffff && heads + 2 * kv_heads <= 65535 * 4,
              "conv_rotary_qk_norm_kv_write: %d / %d heads, %d numbers rotate", heads, kv_heads, rot_dims);
  const int C = (heads + kv_heads) * dim + kv_heads * vdim;
  const auto al16 = [](const void* ptr) { return ((uintptr_t)ptr & 15) == 0; };
  APHRO_CHECK(u_stride >= C && q_out_stride >= (int64_t)heads * dim && u_stride % 8 == 0 && q_out_stride % 8 == 0 && al16(u) && al16(w) && al16(state) &&
                  al16(q_out) && al16(k_cache) && al16(v_cache) && al16(q_weight) && al16(k_weight),
              "conv_rotary_qk_norm_kv_write: rows of 16-byte pieces, aligned");
  int tph = 1;
  while (8 * tph < (dim > vdim ? dim : vdim)) tph *= 2;
  const int units = heads + 2 * kv_heads, per_block = CR_THREADS / tph;
  const bool single = max_q_len == 1;                        // every segment is one token: rows are tiled singly and advance their states
  const int tok = single ? 1 : 4;
  const dim3 grid((unsigned)((num_tokens + tok - 1) / tok), (unsigned)((units + per_block - 1) / per_block));
  const size_t lds = (size_t)8 * CR_THREADS * sizeof(float) + (size_t)tok * (rot_dims / 2) * sizeof(f32x2);
#define CR_LAUNCH(TAPS)                                                                                                               \
  if (single) hipLaunchKernelGGL((conv_rotary_qk_norm_kv_write_kernel<T, TAPS, 1>), grid, dim3(CR_THREADS), lds, (hipStream_t)stream, p); \
  else hipLaunchKernelGGL((conv_rotary_qk_norm_kv_write_kernel<T, TAPS, 4>), grid, dim3(CR_THREADS), lds, (hipStream_t)stream, p)
  MIX_DISPATCH_DTYPE(dtype, {
    typedef typename T::storage S;
    ConvRotaryParams<T> p;
    p.q_out = (S*)q_out; p.k_cache = (S*)k_cache; p.v_cache = (S*)v_cache; p.state = (S*)state;
    p.u = (const S*)u; p.w = (const S*)w; p.q_weight = (const S*)q_weight; p.k_weight = (const S*)k_weight;
    p.slot_mapping = slot_mapping; p.state_slots = state_slots; p.q_start = q_start; p.ctx_len = ctx_len; p.seq_of_token = seq_of_token;
    p.inv_freq = inv_freq; p.q_out_stride = q_out_stride; p.u_stride = u_stride; p.num_cache_rows = num_cache_rows; p.num_tokens = num_tokens;
    p.heads = heads; p.kv_heads = kv_heads; p.dim = dim; p.vdim = vdim; p.rot_dims = rot_dims; p.tph = tph;
    p.write_state = single && taps > 1; p.mscale = mscale; p.eps = eps;
    switch (taps) {
      case 1: CR_LAUNCH(1); break;
      case 2: CR_LAUNCH(2); break;
      case 3: CR_LAUNCH(3); break;
      default: CR_LAUNCH(4); break;
    }
  });
#undef CR_LAUNCH
  APHRO_LAUNCH_CHECK();
  if (single || taps == 1) return APHRO_OK;
  return aphro_short_conv_state(state, u, u_stride, state_slots, q_start, q_len, ctx_len, num_seqs, C, taps, dtype, stream);
}
