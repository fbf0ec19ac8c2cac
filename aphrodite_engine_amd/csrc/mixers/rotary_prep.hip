// What happens between the input product [q | k | v] of a rotary grouped-query attention and its paged cache, in one launch:
//   * the first rot_dims numbers of every query and key head are turned by position * inv_freq[i] -- layout 0 pairs number i
//     with number i + rot_dims / 2 ("rotate half"), layout 1 pairs number 2 i with number 2 i + 1 (interleaved); the pair
//     (u, v) becomes (u cos a - v sin a, v cos a + u sin a), cos and sin times mscale; the rest of the head passes unchanged;
//   * optionally every query and key head is divided by its root mean square over the head, with a weight per number of the
//     head (one for queries, one for keys, shared by their heads) or without.  The weight acts before the rotation; the
//     statistic is taken before it too;
//   * optionally the values are blended with another tensor's values of the same tokens, v <- (1 - lambda) v + lambda v_other;
//   * queries go to a dense output, keys and values into the token-major paged caches at the rows' slots.
// Positions, angles, cos / sin, the statistics and the blend are fp32; one rounding to the storage type.
// One wave per (token, unit): units are the query heads, then the key heads, then the value heads.
//
// qk_row_norm_kv_write is the preparation of an attention whose queries and keys are normed over the WHOLE projection (all heads
// of a token at once, a weight per number) and not rotated: one workgroup per token.
#include "mixers_common.h"

namespace aphro {

template <typename T>
__global__ __launch_bounds__(256) void rotary_qk_norm_kv_write_kernel(
    typename T::storage* __restrict__ q_out, int64_t q_out_stride, typename T::storage* __restrict__ k_cache,
    typename T::storage* __restrict__ v_cache, const int64_t* __restrict__ slot_mapping, int64_t num_cache_rows,
    const typename T::storage* __restrict__ q, int64_t q_stride, const typename T::storage* __restrict__ k, int64_t k_stride,
    const typename T::storage* __restrict__ v, int64_t v_stride, const typename T::storage* __restrict__ v_other,
    int64_t v_other_stride, float lambda, const int32_t* __restrict__ q_start, const int32_t* __restrict__ ctx_len,
    const int32_t* __restrict__ seq_of_token, const float* __restrict__ inv_freq, float mscale, int heads, int kv_heads, int dim, int vdim,
    int rot_dims, int layout, int qk_norm, const typename T::storage* __restrict__ q_weight,
    const typename T::storage* __restrict__ k_weight, float eps) {
  const int64_t t = blockIdx.x;
  const int unit = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (unit >= heads + 2 * kv_heads) return;
  const int64_t slot = slot_mapping[t];
  const bool cached = slot >= 0 && slot < num_cache_rows;
  if (unit >= heads + kv_heads) {                            // a value head
    if (!cached) return;
    const int g = unit - heads - kv_heads;
    const typename T::storage* src = v + t * v_stride + (int64_t)g * vdim;
    typename T::storage* dst = v_cache + (slot * kv_heads + g) * (int64_t)vdim;
    for (int i = lane; i < vdim; i += 64) {
      float x = T::to_f32(src[i]);
      if (v_other) x = (1.0f - lambda) * x + lambda * T::to_f32(v_other[t * v_other_stride + (int64_t)g * vdim + i]);
      dst[i] = T::from_f32(x);
    }
    return;
  }
  const bool is_q = unit < heads;
  if (!is_q && !cached) return;
  const int hd = is_q ? unit : unit - heads;
  const typename T::storage* src = is_q ? q + t * q_stride + (int64_t)hd * dim : k + t * k_stride + (int64_t)hd * dim;
  typename T::storage* dst = is_q ? q_out + t * q_out_stride + (int64_t)hd * dim : k_cache + (slot * kv_heads + hd) * (int64_t)dim;
  const int s = seq_of_token[t];
  const float pos = (float)(ctx_len[s] + (int)(t - q_start[s]));
  const int half = rot_dims >> 1;
  const typename T::storage* nw = is_q ? q_weight : k_weight;
  constexpr int MAXE = 8;                                    // dim <= 512
  float val[MAXE];
  float ss = 0.f;
#pragma unroll
  for (int e = 0; e < MAXE; ++e) {
    const int i = lane + 64 * e;
    float x = 0.f;
    if (i < dim) {
      x = T::to_f32(src[i]);
      ss += x * x;
      if (nw) x *= T::to_f32(nw[i]);
      if (i < 2 * half) {
        int f, partner;
        bool first;
        if (layout == 0) {
          first = i < half;
          f = first ? i : i - half;
          partner = first ? i + half : i - half;
        } else {
          first = (i & 1) == 0;
          f = i >> 1;
          partner = i ^ 1;
        }
        float c, sn;
        sincosf(pos * inv_freq[f], &sn, &c);
        c *= mscale;
        sn *= mscale;
        float other = T::to_f32(src[partner]);
        if (nw) other *= T::to_f32(nw[partner]);
        x = first ? x * c - other * sn : x * c + other * sn;
      }
    }
    val[e] = x;
  }
  float f = 1.0f;
  if (qk_norm) f = 1.0f / sqrtf(wave_sum(ss) / (float)dim + eps);
#pragma unroll
  for (int e = 0; e < MAXE; ++e) {
    const int i = lane + 64 * e;
    if (i < dim) dst[i] = T::from_f32(val[e] * f);
  }
}

template <typename T>
__device__ __forceinline__ void rp_load8(const typename T::storage* p, float* o) {
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
__device__ __forceinline__ void rp_store8(typename T::storage* p, const float* v) {
  if constexpr (sizeof(typename T::storage) == 2) {
    u16x8 r;
#pragma unroll
    for (int j = 0; j < 8; ++j) r[j] = T::from_f32(v[j]);
    *reinterpret_cast<u16x8*>(p) = r;
  } else {
    *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
    *reinterpret_cast<f32x4*>(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
  }
}

// The same for head sizes that are multiples of 8 with 16-byte-aligned rows: a thread owns 8 neighbouring numbers of one unit,
// tph (a power of two, <= 64) threads share a unit, a wave holds 64 / tph units; the rotation partner of a chunk is the chunk
// half the rotated part away (layout 0: rot_dims / 2 is a multiple of 8) or lies within the chunk (layout 1).
template <typename T>
__global__ __launch_bounds__(256) void rotary_qk_norm_kv_write_vec8_kernel(
    typename T::storage* __restrict__ q_out, int64_t q_out_stride, typename T::storage* __restrict__ k_cache,
    typename T::storage* __restrict__ v_cache, const int64_t* __restrict__ slot_mapping, int64_t num_cache_rows,
    const typename T::storage* __restrict__ q, int64_t q_stride, const typename T::storage* __restrict__ k, int64_t k_stride,
    const typename T::storage* __restrict__ v, int64_t v_stride, const typename T::storage* __restrict__ v_other,
    int64_t v_other_stride, float lambda, const int32_t* __restrict__ q_start, const int32_t* __restrict__ ctx_len,
    const int32_t* __restrict__ seq_of_token, const float* __restrict__ inv_freq, float mscale, int heads, int kv_heads, int dim, int vdim,
    int rot_dims, int layout, int qk_norm, const typename T::storage* __restrict__ q_weight,
    const typename T::storage* __restrict__ k_weight, float eps, int tph) {
  const int64_t t = blockIdx.x;
  const int per_block = 256 / tph;
  const int unit = blockIdx.y * per_block + threadIdx.x / tph, i0 = 8 * (threadIdx.x % tph);
  const bool live = unit < heads + 2 * kv_heads;          // every lane stays for the shuffles below
  const int64_t slot = slot_mapping[t];
  const bool cached = slot >= 0 && slot < num_cache_rows;
  if (live && unit >= heads + kv_heads) {                   // a value head
    const int g = unit - heads - kv_heads;
    if (cached && i0 < vdim) {
      float x[8];
      rp_load8<T>(v + t * v_stride + (int64_t)g * vdim + i0, x);
      if (v_other) {
        float o[8];
        rp_load8<T>(v_other + t * v_other_stride + (int64_t)g * vdim + i0, o);
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = (1.0f - lambda) * x[e] + lambda * o[e];
      }
      rp_store8<T>(v_cache + (slot * kv_heads + g) * (int64_t)vdim + i0, x);
    }
  }
  const bool qk = live && unit < heads + kv_heads;
  const bool is_q = unit < heads;
  const int hd = is_q ? unit : unit - heads;
  const bool work = qk && i0 < dim && (is_q || cached);
  float x[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) x[e] = 0.f;
  float ss = 0.f;
  if (work) {
    const typename T::storage* src = is_q ? q + t * q_stride + (int64_t)hd * dim : k + t * k_stride + (int64_t)hd * dim;
    rp_load8<T>(src + i0, x);
    const typename T::storage* nw = is_q ? q_weight : k_weight;
#pragma unroll
    for (int e = 0; e < 8; ++e) ss += x[e] * x[e];
    if (nw) {
      float w[8];
      rp_load8<T>(nw + i0, w);
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] *= w[e];
    }
    if (i0 < rot_dims) {
      const int s = seq_of_token[t];
      const float pos = (float)(ctx_len[s] + (int)(t - q_start[s]));
      const int half = rot_dims >> 1;
      if (layout == 0) {
        const bool first = i0 < half;
        float o[8];
        rp_load8<T>(src + (first ? i0 + half : i0 - half), o);
        if (nw) {
          float w[8];
          rp_load8<T>(nw + (first ? i0 + half : i0 - half), w);
#pragma unroll
          for (int e = 0; e < 8; ++e) o[e] *= w[e];
        }
        const int f0 = first ? i0 : i0 - half;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          float c, sn;
          sincosf(pos * inv_freq[f0 + e], &sn, &c);
          c *= mscale;
          sn *= mscale;
          x[e] = first ? x[e] * c - o[e] * sn : x[e] * c + o[e] * sn;
        }
      } else {
#pragma unroll
        for (int e = 0; e < 8; e += 2) {
          float c, sn;
          sincosf(pos * inv_freq[(i0 + e) >> 1], &sn, &c);
          c *= mscale;
          sn *= mscale;
          const float a = x[e], b = x[e + 1];
          x[e] = a * c - b * sn;
          x[e + 1] = b * c + a * sn;
        }
      }
    }
  }
  float f = 1.0f;
  if (qk_norm) {
    for (int o = tph >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
    f = 1.0f / sqrtf(ss / (float)dim + eps);
  }
  if (work) {
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] *= f;
    typename T::storage* dst = is_q ? q_out + t * q_out_stride + (int64_t)hd * dim : k_cache + (slot * kv_heads + hd) * (int64_t)dim;
    rp_store8<T>(dst + i0, x);
  }
}

// A row of n numbers times 1 / rms(row) times weight, from src to dst; CH chunks of 8 per thread stay in registers (CH 0: any
// size and alignment, the row is read twice).
template <typename T, int CH>
__device__ __forceinline__ void row_norm(typename T::storage* dst, const typename T::storage* src, const typename T::storage* weight,
                                         int n, float eps, float* red) {
  float ss = 0.f;
  if constexpr (CH == 0) {
    for (int i = threadIdx.x; i < n; i += blockDim.x) {
      const float x = T::to_f32(src[i]);
      ss += x * x;
    }
    const float f = 1.0f / sqrtf(wg_sum(ss, red) / (float)n + eps);
    if (dst)
      for (int i = threadIdx.x; i < n; i += blockDim.x) dst[i] = T::from_f32(T::to_f32(src[i]) * f * T::to_f32(weight[i]));
  } else {
    float x[CH][8];
#pragma unroll
    for (int c = 0; c < CH; ++c) {
      const int i0 = (threadIdx.x + c * blockDim.x) * 8;
      if (i0 < n) {
        rp_load8<T>(src + i0, x[c]);
#pragma unroll
        for (int e = 0; e < 8; ++e) ss += x[c][e] * x[c][e];
      }
    }
    const float f = 1.0f / sqrtf(wg_sum(ss, red) / (float)n + eps);
    if (dst) {
#pragma unroll
      for (int c = 0; c < CH; ++c) {
        const int i0 = (threadIdx.x + c * blockDim.x) * 8;
        if (i0 < n) {
          float w[8];
          rp_load8<T>(weight + i0, w);
#pragma unroll
          for (int e = 0; e < 8; ++e) x[c][e] = x[c][e] * f * w[e];
          rp_store8<T>(dst + i0, x[c]);
        }
      }
    }
  }
}

// blockIdx.y 0: the query row; 1: the key row and the values.
template <typename T, int CH>
__global__ __launch_bounds__(256) void qk_row_norm_kv_write_kernel(
    typename T::storage* __restrict__ q_out, int64_t q_out_stride, typename T::storage* __restrict__ k_cache,
    typename T::storage* __restrict__ v_cache, const int64_t* __restrict__ slot_mapping, int64_t num_cache_rows,
    const typename T::storage* __restrict__ q, int64_t q_stride, const typename T::storage* __restrict__ k, int64_t k_stride,
    const typename T::storage* __restrict__ v, int64_t v_stride, const typename T::storage* __restrict__ q_weight,
    const typename T::storage* __restrict__ k_weight, int nq, int nk, int nv, float eps) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  if (blockIdx.y == 0) {
    row_norm<T, CH>(q_out + t * q_out_stride, q + t * q_stride, q_weight, nq, eps, red);
    return;
  }
  const int64_t slot = slot_mapping[t];
  const bool cached = slot >= 0 && slot < num_cache_rows;
  row_norm<T, CH>(cached ? k_cache + slot * nk : nullptr, k + t * k_stride, k_weight, nk, eps, red);
  if (!cached) return;
  const typename T::storage* src = v + t * v_stride;
  typename T::storage* dst = v_cache + slot * nv;
  if constexpr (CH == 0) {
    for (int i = threadIdx.x; i < nv; i += blockDim.x) dst[i] = src[i];
  } else {
    for (int i0 = threadIdx.x * 8; i0 < nv; i0 += blockDim.x * 8) {
      float x[8];
      rp_load8<T>(src + i0, x);
      rp_store8<T>(dst + i0, x);
    }
  }
}

}  // namespace aphro

using namespace aphro;

extern "C" int aphro_rotary_qk_norm_kv_write(void* q_out, int64_t q_out_stride, void* k_cache, void* v_cache, const int64_t* slot_mapping,
                                             int64_t num_cache_rows, const void* q, int64_t q_stride, const void* k, int64_t k_stride,
                                             const void* v, int64_t v_stride, const void* v_other, int64_t v_other_stride, float lambda,
                                             const int32_t* q_start, const int32_t* ctx_len, const int32_t* seq_of_token,
                                             const float* inv_freq, float mscale, int64_t num_tokens, int heads, int kv_heads, int dim, int vdim,
                                             int rot_dims, int layout, int qk_norm, const void* q_weight, const void* k_weight, float eps, int dtype, void* stream) {
  if (num_tokens == 0) return APHRO_OK;
  APHRO_CHECK(q_out && k_cache && v_cache && slot_mapping && q && k && v && q_start && ctx_len && seq_of_token && (rot_dims == 0 || inv_freq),
              "rotary_qk_norm_kv_write: null argument");
  APHRO_CHECK(heads > 0 && kv_heads > 0 && dim > 0 && dim <= 512 && vdim > 0 && rot_dims >= 0 && rot_dims <= dim && rot_dims % 2 == 0 &&
                  (layout == 0 || layout == 1) && heads + 2 * kv_heads <= 4 * 65535,
              "rotary_qk_norm_kv_write: %d / %d heads of %d (<= 512) and %d, %d numbers rotate", heads, kv_heads, dim, vdim, rot_dims);
  APHRO_CHECK(q_stride >= (int64_t)heads * dim && q_out_stride >= (int64_t)heads * dim && k_stride >= (int64_t)kv_heads * dim &&
                  v_stride >= (int64_t)kv_heads * vdim && (!v_other || v_other_stride >= (int64_t)kv_heads * vdim) && num_cache_rows > 0,
              "rotary_qk_norm_kv_write: row strides smaller than the rows");
  APHRO_CHECK((q_weight == nullptr) == (k_weight == nullptr) && (!q_weight || qk_norm), "rotary_qk_norm_kv_write: weights belong to the norm, both or none");
  const int units = heads + 2 * kv_heads;
  const auto al16 = [](const void* ptr) { return ((uintptr_t)ptr & 15) == 0; };
  int tph = 1;
  while (8 * tph < (dim > vdim ? dim : vdim)) tph *= 2;
  const bool vec = dim % 8 == 0 && vdim % 8 == 0 && tph <= 64 && (layout == 1 || (rot_dims / 2) % 8 == 0) && rot_dims % 8 == 0 &&
                   q_stride % 8 == 0 && k_stride % 8 == 0 && v_stride % 8 == 0 && q_out_stride % 8 == 0 && v_other_stride % 8 == 0 &&
                   al16(q) && al16(k) && al16(v) && al16(v_other) && al16(q_out) && al16(k_cache) && al16(v_cache) &&
                   al16(q_weight) && al16(k_weight);
  MIX_DISPATCH_DTYPE(dtype, {
    typedef typename T::storage S;
    if (vec) {
      const int per_block = 256 / tph;
      hipLaunchKernelGGL((rotary_qk_norm_kv_write_vec8_kernel<T>), dim3((unsigned)num_tokens, (unsigned)((units + per_block - 1) / per_block)),
                         dim3(256), 0, (hipStream_t)stream, (S*)q_out, q_out_stride, (S*)k_cache, (S*)v_cache, slot_mapping, num_cache_rows,
                         (const S*)q, q_stride, (const S*)k, k_stride, (const S*)v, v_stride, (const S*)v_other, v_other_stride, lambda,
                         q_start, ctx_len, seq_of_token, inv_freq, mscale, heads, kv_heads, dim, vdim, rot_dims, layout, qk_norm,
                         (const S*)q_weight, (const S*)k_weight, eps, tph);
    } else
    hipLaunchKernelGGL((rotary_qk_norm_kv_write_kernel<T>), dim3((unsigned)num_tokens, (unsigned)((units + 3) / 4)), dim3(256), 0,
                       (hipStream_t)stream, (S*)q_out, q_out_stride, (S*)k_cache, (S*)v_cache, slot_mapping, num_cache_rows, (const S*)q,
                       q_stride, (const S*)k, k_stride, (const S*)v, v_stride, (const S*)v_other, v_other_stride, lambda, q_start,
                       ctx_len, seq_of_token, inv_freq, mscale, heads, kv_heads, dim, vdim, rot_dims, layout, qk_norm, (const S*)q_weight,
                       (const S*)k_weight, eps);
  });
  APHRO_LAUNCH_CHECK();
  return APHRO_OK;
}

extern "C" int aphro_qk_row_norm_kv_write(void* q_out, int64_t q_out_stride, void* k_cache, void* v_cache, const int64_t* slot_mapping,
                                          int64_t num_cache_rows, const void* q, int64_t q_stride, const void* k, int64_t k_stride,
                                          const void* v, int64_t v_stride, const void* q_weight, const void* k_weight,
                                          int64_t num_tokens, int nq, int nk, int nv, float eps, int dtype, void* stream) {
  if (num_tokens == 0) return APHRO_OK;
  APHRO_CHECK(q_out && k_cache && v_cache && slot_mapping && q && k && v && q_weight && k_weight, "qk_row_norm_kv_write: null argument");
  APHRO_CHECK(nq > 0 && nk > 0 && nv > 0 && q_stride >= nq && q_out_stride >= nq && k_stride >= nk && v_stride >= nv && num_cache_rows > 0,
              "qk_row_norm_kv_write: rows of %d / %d / %d", nq, nk, nv);
  const auto al16 = [](const void* ptr) { return ((uintptr_t)ptr & 15) == 0; };
  const bool vec = nq % 8 == 0 && nk % 8 == 0 && nv % 8 == 0 && q_stride % 8 == 0 && k_stride % 8 == 0 && v_stride % 8 == 0 &&
                   q_out_stride % 8 == 0 && al16(q) && al16(k) && al16(v) && al16(q_out) && al16(k_cache) && al16(v_cache) &&
                   al16(q_weight) && al16(k_weight);
  const int longest = nq > nk ? nq : nk;
  const dim3 grid((unsigned)num_tokens, 2u);
  int threads = 256;
  if (vec && longest <= 8 * 256) threads = (longest / 8 + 63) / 64 * 64;
#define QKR_LAUNCH(CH)                                                                                                              \
  hipLaunchKernelGGL((qk_row_norm_kv_write_kernel<T, CH>), grid, dim3(threads), 0, (hipStream_t)stream, (S*)q_out, q_out_stride,     \
                     (S*)k_cache, (S*)v_cache, slot_mapping, num_cache_rows, (const S*)q, q_stride, (const S*)k, k_stride,           \
                     (const S*)v, v_stride, (const S*)q_weight, (const S*)k_weight, nq, nk, nv, eps)
  MIX_DISPATCH_DTYPE(dtype, {
    typedef typename T::storage S;
    if (vec && longest <= 8 * 256) QKR_LAUNCH(1);
    else if (vec && longest <= 16 * 256) QKR_LAUNCH(2);
    else if (vec && longest <= 32 * 256) QKR_LAUNCH(4);
    else QKR_LAUNCH(0);
  });
#undef QKR_LAUNCH
  APHRO_LAUNCH_CHECK();
  return APHRO_OK;
}
