// A bounded elementwise map in the place of a norm, tanh(alpha * x) * weight + bias, around the
// float32 residual stream: the kernel first adds what is pending, x <- x + scale * delta (a tensor of
// the compute dtype, or the float32 partial sums of a split product, added in order), stores the
// stream and leaves the mapped rows in the compute dtype.  Nothing is reduced over a row, so
// threads take runs of four elements wherever they lie.  Without an output it only adds.
#include "api.h"
#include "common.h"

namespace shk {

namespace {

constexpr int kDytThreads = 256;
constexpr int kDytParts = 4;  // parts of a split product in flight

template <typename T, int V>
__device__ __forceinline__ void dyt_load(const T* p, float (&x)[V]) {
  if constexpr (V == 1) {
    x[0] = to_float(p[0]);
  } else if constexpr (sizeof(T) == 4) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    x[0] = a.x, x[1] = a.y, x[2] = a.z, x[3] = a.w;
  } else {
    const uint2 u = *reinterpret_cast<const uint2*>(p);
    x[0] = __uint_as_float(u.x << 16), x[1] = __uint_as_float(u.x & 0xffff0000u);
    x[2] = __uint_as_float(u.y << 16), x[3] = __uint_as_float(u.y & 0xffff0000u);
  }
}

template <typename T, int V>
__device__ __forceinline__ void dyt_store(T* p, const float (&x)[V]) {
  if constexpr (V == 1) {
    p[0] = from_float<T>(x[0]);
  } else if constexpr (sizeof(T) == 4) {
    *reinterpret_cast<float4*>(p) = make_float4(x[0], x[1], x[2], x[3]);
  } else {
    uint2 u;
    u.x = bf16_bits(x[0]) | (static_cast<uint32_t>(bf16_bits(x[1])) << 16);
    u.y = bf16_bits(x[2]) | (static_cast<uint32_t>(bf16_bits(x[3])) << 16);
    *reinterpret_cast<uint2*>(p) = u;
  }
}

// T: the compute dtype; TD: the type of delta, T, or float for partial sums
template <typename T, typename TD, int V>
__global__ void __launch_bounds__(kDytThreads)
    add_dynamic_tanh_kernel(float* __restrict__ resid, const TD* __restrict__ delta, int splits, size_t split_stride,
                            float scale, float alpha, const float* __restrict__ weight, const float* __restrict__ bias,
                            T* __restrict__ out, const int32_t* __restrict__ rows, int n, int hidden, int write_resid) {
  const int per_row = hidden / V;
  const long long i = static_cast<long long>(blockIdx.x) * kDytThreads + threadIdx.x;
  if (i >= static_cast<long long>(n) * per_row) return;
  const int r = static_cast<int>(i / per_row), c = static_cast<int>(i % per_row) * V;
  const size_t at = (rows ? static_cast<size_t>(rows[r]) : static_cast<size_t>(r)) * hidden + c;
  float x[V], d[V], w[V], b[V];
  dyt_load<float, V>(resid + at, x);
  if (out) {
    dyt_load<float, V>(weight + c, w);
    dyt_load<float, V>(bias + c, b);
  }
  if (delta) {
    dyt_load<TD, V>(delta + at, d);
    for (int z0 = 1; z0 < splits; z0 += kDytParts) {  // further parts, added in order
      float more[kDytParts][V];
#pragma unroll
      for (int u = 0; u < kDytParts; ++u)
        dyt_load<TD, V>(delta + static_cast<size_t>(z0 + u < splits ? z0 + u : splits - 1) * split_stride + at, more[u]);
#pragma unroll
      for (int u = 0; u < kDytParts; ++u)
        if (z0 + u < splits) {
#pragma unroll
          for (int e = 0; e < V; ++e) d[e] += more[u][e];
        }
    }
#pragma unroll
    for (int e = 0; e < V; ++e) x[e] = fmaf(scale, d[e], x[e]);
    if (write_resid) dyt_store<float, V>(resid + at, x);
  }
  if (!out) return;
  float y[V];
#pragma unroll
  for (int e = 0; e < V; ++e) y[e] = fmaf(tanhf(alpha * x[e]), w[e], b[e]);
  dyt_store<T, V>(out + static_cast<size_t>(r) * hidden + c, y);
}

}  // namespace

}  // namespace shk

using namespace shk;

extern "C" int shk_add_dynamic_tanh(float* resid, const void* delta, int delta_splits, float scale, float alpha,
                                    const float* weight, const float* bias, void* out, int dtype, const int32_t* rows,
                                    int n, int hidden, int write_resid, int resid_rows, void* stream) {
  SHK_REQUIRE(dtype == kF32 || dtype == kBF16, "add_dynamic_tanh: unknown dtype %d", dtype);
  SHK_REQUIRE(n >= 0 && hidden > 0 && delta_splits >= 0 && resid_rows >= 0, "add_dynamic_tanh: bad sizes n=%d hidden=%d",
              n, hidden);
  if (n == 0) return 0;
  SHK_REQUIRE(resid && (!out || (weight && bias)), "add_dynamic_tanh: null pointer");
  SHK_REQUIRE(out || (delta && write_resid), "add_dynamic_tanh: nothing to write");
  SHK_REQUIRE(delta || delta_splits == 0, "add_dynamic_tanh: partial sums without a pointer");
  hipStream_t s = static_cast<hipStream_t>(stream);
  const size_t stride = static_cast<size_t>(resid_rows) * hidden;
  bool four = hidden % 4 == 0;
  for (const void* p : {static_cast<const void*>(resid), delta, static_cast<const void*>(weight),
                        static_cast<const void*>(bias), static_cast<const void*>(out)})
    four = four && reinterpret_cast<uintptr_t>(p) % 16 == 0;
  const long long items = static_cast<long long>(n) * (hidden / (four ? 4 : 1));
  SHK_REQUIRE(items < (1LL << 31) * kDytThreads, "add_dynamic_tanh: too many elements");
  const unsigned grid = static_cast<unsigned>((items + kDytThreads - 1) / kDytThreads);
#define SHK_GO(T, TD, V)                                                                                             \
  add_dynamic_tanh_kernel<T, TD, V><<<grid, kDytThreads, 0, s>>>(resid, static_cast<const TD*>(delta), delta_splits, \
                                                                 stride, scale, alpha, weight, bias,                 \
                                                                 static_cast<T*>(out), rows, n, hidden, write_resid)
#define SHK_V(T, TD)                            \
  do {                                          \
    if (four) SHK_GO(T, TD, 4);                 \
    else SHK_GO(T, TD, 1);                      \
  } while (0)
  if (dtype == kF32) SHK_V(float, float);
  else if (delta_splits > 0) SHK_V(bf16, float);
  else SHK_V(bf16, bf16);
#undef SHK_V
#undef SHK_GO
  SHK_LAUNCH_CHECK("add_dynamic_tanh");
  return 0;
}
