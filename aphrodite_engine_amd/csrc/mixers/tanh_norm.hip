// The launch between the layers of a decoder whose norm is a dynamic tanh -- norm(x) = tanh(alpha x) w + b, elementwise, no statistic
// of the row -- around an fp32 residual stream:
//   r = x + y_a + y_b + table[ids[t]]        every term optional; `fresh`: x is not read (the stream starts here)
//   x = r;   out_1 = norm_1(r),  out_2 = norm_2(r)       each optional
// One launch so joins the results of the sublayers that ran side by side, adds an embedding row (the start of the stream, or the
// embedding output once more ahead of a repeated span of layers) and rounds the inputs of the next layer's sublayers, which have a
// norm each.  All fp32; one rounding to the storage type.  Rows that are a multiple of 8 and 16-byte aligned: 8 elements per thread.
#include "mixers_common.h"

namespace aphro {

template <typename T>
struct TanhNorm {
  const typename T::storage* w;
  const typename T::storage* b;
  typename T::storage* out;       // NULL: this norm is not asked for
  float alpha;
};

template <typename T>
__device__ __forceinline__ void tn_load8(const typename T::storage* p, float* o) {
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
__device__ __forceinline__ void tn_store8(typename T::storage* p, const float* v) {
  if constexpr (sizeof(typename T::storage) == 2) {
    *reinterpret_cast<u32x4*>(p) = u32x4{pack2_16<true>(v[0], v[1]), pack2_16<true>(v[2], v[3]), pack2_16<true>(v[4], v[5]), pack2_16<true>(v[6], v[7])};
  } else {
    *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
    *reinterpret_cast<f32x4*>(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
  }
}

template <typename T>
__device__ __forceinline__ void tanh_norm8(const TanhNorm<T>& n, const float* r, int i0, int64_t at) {
  if (n.out == nullptr) return;
  float w[8], b[8];
  tn_load8<T>(n.w + i0, w);
  tn_load8<T>(n.b + i0, b);
#pragma unroll
  for (int j = 0; j < 8; ++j) w[j] = tanhf(n.alpha * r[j]) * w[j] + b[j];
  tn_store8<T>(n.out + at, w);
}

template <typename T>
__global__ __launch_bounds__(256) void residual_tanh_norm_vec8_kernel(float* __restrict__ x, int fresh, const typename T::storage* __restrict__ ya,
                                                                      int64_t ya_stride, const typename T::storage* __restrict__ yb,
                                                                      int64_t yb_stride, const typename T::storage* __restrict__ table,
                                                                      const int64_t* __restrict__ ids, int64_t vocab, TanhNorm<T> n1,
                                                                      TanhNorm<T> n2, int width) {
  const int64_t t = blockIdx.x;
  const int i0 = (blockIdx.y * blockDim.x + threadIdx.x) * 8;
  if (i0 >= width) return;
  const int64_t at = t * (int64_t)width + i0;
  float r[8];
  if (fresh) {
#pragma unroll
    for (int j = 0; j < 8; ++j) r[j] = 0.f;
  } else {
    tn_load8<Float>(x + at, r);
  }
  float y[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) y[j] = 0.f;
  if (ya) tn_load8<T>(ya + t * ya_stride + i0, y);
  if (yb) {
    float z[8];
    tn_load8<T>(yb + t * yb_stride + i0, z);
#pragma unroll
    for (int j = 0; j < 8; ++j) y[j] += z[j];
  }
#pragma unroll
  for (int j = 0; j < 8; ++j) r[j] += y[j];
  if (table) {
    int64_t id = ids[t];
    if (id < 0 || id >= vocab) id = 0;
    float e[8];
    tn_load8<T>(table + id * (int64_t)width + i0, e);
#pragma unroll
    for (int j = 0; j < 8; ++j) r[j] += e[j];
  }
  if (fresh || ya || yb || table) tn_store8<Float>(x + at, r);
  tanh_norm8<T>(n1, r, i0, at);
  tanh_norm8<T>(n2, r, i0, at);
}

template <typename T>
__global__ __launch_bounds__(256) void residual_tanh_norm_kernel(float* __restrict__ x, int fresh, const typename T::storage* __restrict__ ya,
                                                                 int64_t ya_stride, const typename T::storage* __restrict__ yb,
                                                                 int64_t yb_stride, const typename T::storage* __restrict__ table,
                                                                 const int64_t* __restrict__ ids, int64_t vocab, TanhNorm<T> n1, TanhNorm<T> n2,
                                                                 int width) {
  const int64_t t = blockIdx.x;
  const int i = blockIdx.y * blockDim.x + threadIdx.x;
  if (i >= width) return;
  const int64_t at = t * (int64_t)width + i;
  float r = fresh ? 0.f : x[at], y = ya ? T::to_f32(ya[t * ya_stride + i]) : 0.f;
  if (yb) y += T::to_f32(yb[t * yb_stride + i]);
  r += y;
  if (table) {
    int64_t id = ids[t];
    if (id < 0 || id >= vocab) id = 0;
    r += T::to_f32(table[id * (int64_t)width + i]);
  }
  if (fresh || ya || yb || table) x[at] = r;
  if (n1.out) n1.out[at] = T::from_f32(tanhf(n1.alpha * r) * T::to_f32(n1.w[i]) + T::to_f32(n1.b[i]));
  if (n2.out) n2.out[at] = T::from_f32(tanhf(n2.alpha * r) * T::to_f32(n2.w[i]) + T::to_f32(n2.b[i]));
}

}  // namespace aphro

using namespace aphro;

extern "C" int aphro_residual_tanh_norm(float* x, int fresh, const void* ya, int64_t ya_stride, const void* yb, int64_t yb_stride,
                                        const void* table, const int64_t* ids, int64_t vocab, float alpha1, const void* w1, const void* b1,
                                        void* out1, float alpha2, const void* w2, const void* b2, void* out2, int64_t num_tokens, int width,
                                        int dtype, void* stream) {
  if (num_tokens == 0) return APHRO_OK;
  APHRO_CHECK(x && num_tokens > 0 && num_tokens <= 0x7fffffff && width > 0 && width <= 256 * 65535, "residual_tanh_norm: bad sizes (width %d)", width);
  APHRO_CHECK((!ya || ya_stride >= width) && (!yb || yb_stride >= width), "residual_tanh_norm: a row stride is smaller than the row");
  APHRO_CHECK(!table || (ids && vocab > 0), "residual_tanh_norm: a table needs the rows' ids");
  APHRO_CHECK((!out1 || (w1 && b1)) && (!out2 || (w2 && b2)), "residual_tanh_norm: a norm needs its weight and bias");
  APHRO_CHECK(fresh || ya || yb || table || out1 || out2, "residual_tanh_norm: nothing to do");
  const auto al16 = [](const void* ptr) { return ((uintptr_t)ptr & 15) == 0; };
  const bool vec = (width & 7) == 0 && (ya_stride & 7) == 0 && (yb_stride & 7) == 0 && al16(x) && al16(ya) && al16(yb) && al16(table) &&
                   al16(w1) && al16(b1) && al16(out1) && al16(w2) && al16(b2) && al16(out2);
  const int units = vec ? width / 8 : width;
  // narrow workgroups while there are few of them (decoded rows), so that the launch covers the chip
  const int most = num_tokens * ((units + 255) / 256) < 512 ? 64 : 256;
  const int threads = units >= most ? most : (units + 63) / 64 * 64;
  const dim3 grid((unsigned)num_tokens, (unsigned)((units + threads - 1) / threads));
  MIX_DISPATCH_DTYPE(dtype, {
    typedef typename T::storage S;
    const TanhNorm<T> n1 = {(const S*)w1, (const S*)b1, (S*)out1, alpha1}, n2 = {(const S*)w2, (const S*)b2, (S*)out2, alpha2};
    if (vec)
      hipLaunchKernelGGL((residual_tanh_norm_vec8_kernel<T>), grid, dim3(threads), 0, (hipStream_t)stream, x, fresh, (const S*)ya, ya_stride,
                         (const S*)yb, yb_stride, (const S*)table, ids, vocab, n1, n2, width);
    else
      hipLaunchKernelGGL((residual_tanh_norm_kernel<T>), grid, dim3(threads), 0, (hipStream_t)stream, x, fresh, (const S*)ya, ya_stride,
                         (const S*)yb, yb_stride, (const S*)table, ids, vocab, n1, n2, width);
  });
  APHRO_LAUNCH_CHECK();
  return APHRO_OK;
}
