// The real-gated linear recurrent unit (Griffin), per channel c:
//   r = sigmoid(zr + br),  i = sigmoid(zi + bi),  log a = -rate_c r,  a = exp(log a)
//   S_t = a S_(t-1) + sqrt(1 - a^2) i u_t;   out_t = S_t gelu(y_t)      (tanh form of GELU)
// zr and zi are the gates' products (float32) before their biases, rate_c a positive number per
// channel, u the convolved input, y the other branch's projection.  All of it and the state are
// float32.  A request's slot holds S [width] and then the convolution's last taps - 1 inputs
// [(taps - 1), width], oldest first; a state counts as zero where the sequence's first row of the
// step is at position 0.
//
// Single tokens: a thread per channel.  Prompt portions: a workgroup of 16 wavefronts owns 16
// channels of a sequence and walks its tokens in tiles of 512; the quarters of a wavefront take 8
// tokens each.  (Workgroups with neighbouring channels run on one XCD, whose L2 then serves both
// halves of a line.)  What does not depend on the state (gates, exponentials, roots) is formed for
// all tokens of a tile at once, the next tile's inputs are on their way meanwhile, and only the
// multiply-adds of S pass from run to run, through lane permutations within a wavefront and through
// LDS and a barrier between wavefronts.  Every token is one multiply-add on the S before it, in
// order, so a result does not depend on how a prompt was cut.
#include "api.h"
#include "common.h"

namespace shk {

namespace {

constexpr int kChannels = 16;   // channels a workgroup of the prompt kernel
constexpr int kRunTokens = 8;   // tokens a lane takes of a tile
constexpr int kGroups = 64;     // runs of tokens a tile: 16 wavefronts of four quarters
constexpr int kQuarters = kWave / kChannels;  // runs of tokens a wavefront
constexpr int kXcds = 8;
constexpr int kTile = kRunTokens * kGroups;

// (bfloat16 models: the hardware's exponential, float32 all the same; float32 models: the library's)
template <typename T>
__device__ __forceinline__ float exp_f(float x) {
  return sizeof(T) == 2 ? __expf(x) : expf(x);
}
template <typename T>
__device__ __forceinline__ float sigmoid_f(float z) {
  return 1.f / (1.f + exp_f<T>(-z));
}
template <typename T>
__device__ __forceinline__ float gelu_f(float z) {
  const float u = 0.7978845608028654f * (z + 0.044715f * z * z * z);
  return z / (1.f + exp_f<T>(-2.f * u));
}

// 1 - a^2 for a = exp(-x / 2): below 1/4 the series x - x^2 / 2! + x^3 / 3! - ... (what is left out is less than
// 2^-24 of the sum), where 1 - a a would lose what a small rate leaves
__device__ __forceinline__ float one_less_square(float x, float a) {
  const float series = x * (1.f - x * (1.f / 2) * (1.f - x * (1.f / 3) * (1.f - x * (1.f / 4) * (1.f - x * (1.f / 5) * (1.f - x * (1.f / 6))))));
  return x < 0.25f ? series : 1.f - a * a;
}

struct Step {
  float a, x;  // S <- a S + x
};
template <typename T>
__device__ __forceinline__ Step make_step(float zr, float zi, float u, float br, float bi, float rate) {
  const float less = rate * sigmoid_f<T>(zr + br);
  Step s;
  s.a = exp_f<T>(-less);
  s.x = sqrtf(one_less_square(2.f * less, s.a)) * (sigmoid_f<T>(zi + bi) * u);
  return s;
}

// The convolution's kept inputs: the taps - 1 positions before the next step, oldest first.  (e + count is
// the old place of the input that moves to e: never one that has been overwritten.)
template <typename T>
__device__ __forceinline__ void keep_tail(float* tail, const T* raw, int ld_raw, int c, int width, int taps, int first,
                                          int last, bool fresh) {
  const int count = last - first;
  for (int e = 0; e < taps - 1; ++e) {
    const int back = taps - 1 - e;
    float v = 0.f;
    if (back <= count)
      v = to_float(raw[static_cast<size_t>(last - back) * ld_raw + c]);
    else if (!fresh)
      v = tail[static_cast<size_t>(e + count) * width + c];
    tail[static_cast<size_t>(e) * width + c] = v;
  }
}

// Column of channel c's zr in a row of the gates' products: block by block [r | i]; zi lies `part` further.
__device__ __forceinline__ int gate_column(int c, int part) { return c / part * 2 * part + c % part; }

template <typename T>
__global__ void __launch_bounds__(256)
    rglru_step_kernel(const float* __restrict__ gates, int part, const float* __restrict__ br,
                      const float* __restrict__ bi, const float* __restrict__ rate, const T* __restrict__ u,
                      const T* __restrict__ y, int ldy, const T* __restrict__ raw, int ld_raw, int width, int taps,
                      const int32_t* __restrict__ positions, const int32_t* __restrict__ cu_q,
                      const int32_t* __restrict__ slots, float* __restrict__ state, long long slot_stride,
                      T* __restrict__ out) {
  const int seq = blockIdx.y;
  const int c = blockIdx.x * 256 + threadIdx.x;
  const int first = cu_q[seq], last = cu_q[seq + 1];
  if (c >= width || last <= first) return;
  const bool fresh = positions[first] == 0;
  float* slot = state + static_cast<size_t>(slots[seq]) * slot_stride;
  float S = fresh ? 0.f : slot[c];
  const float b_r = br[c], b_i = bi[c], rt = rate[c];
  const int col = gate_column(c, part);
  for (int t = first; t < last; ++t) {
    const float* z = gates + static_cast<size_t>(t) * 2 * width + col;
    const Step s = make_step<T>(z[0], z[part], to_float(u[static_cast<size_t>(t) * width + c]), b_r, b_i, rt);
    S = fmaf(s.a, S, s.x);
    out[static_cast<size_t>(t) * width + c] = from_float<T>(S * gelu_f<T>(to_float(y[static_cast<size_t>(t) * ldy + c])));
  }
  slot[c] = S;
  keep_tail(slot + width, raw, ld_raw, c, width, taps, first, last, fresh);
}

// workgroups a sequence: as many on every XCD
inline int blocks_of(int width) {
  const int blocks = (width + kChannels - 1) / kChannels;
  return (blocks + kXcds - 1) / kXcds * kXcds;
}

template <typename T>
__global__ void __launch_bounds__(16 * kWave)
    rglru_scan_kernel(const float* __restrict__ gates, int part, const float* __restrict__ br,
                      const float* __restrict__ bi, const float* __restrict__ rate, const T* __restrict__ u,
                      const T* __restrict__ y, int ldy, const T* __restrict__ raw, int ld_raw, int width, int taps,
                      int first_seq, const int32_t* __restrict__ positions, const int32_t* __restrict__ cu_q,
                      const int32_t* __restrict__ slots, float* __restrict__ state, long long slot_stride,
                      T* __restrict__ out) {
  __shared__ float carry[kChannels];
  const int seq = first_seq + blockIdx.y;
  const int first = cu_q[seq], last = cu_q[seq + 1];
  if (last <= first) return;
  const int group = threadIdx.x / kChannels;  // this thread's run of tokens within a tile
  const int per_xcd = gridDim.x / kXcds;  // (workgroups go to the XCDs in turn)
  const int c_raw = (blockIdx.x % kXcds * per_xcd + blockIdx.x / kXcds) * kChannels + threadIdx.x % kChannels;
  if (c_raw - threadIdx.x % kChannels >= width) return;
  const bool active = c_raw < width;
  const int c = active ? c_raw : width - 1;
  const bool fresh = positions[first] == 0;
  float* slot = state + static_cast<size_t>(slots[seq]) * slot_stride;
  const float b_r = br[c], b_i = bi[c], rt = rate[c];
  const int col = gate_column(c, part);
  if (threadIdx.x < kChannels) carry[threadIdx.x] = fresh ? 0.f : slot[c];

  float zr[kRunTokens], zi[kRunTokens];
  T uv[kRunTokens], yv[kRunTokens];
  auto fetch = [&](int t0) {  // (tokens behind the portion read its last one)
#pragma unroll
    for (int i = 0; i < kRunTokens; ++i) {
      const int tr = t0 + group * kRunTokens + i;
      const size_t t = tr < last ? tr : last - 1;
      zr[i] = gates[t * 2 * width + col];
      zi[i] = gates[t * 2 * width + col + part];
      uv[i] = u[t * width + c];
      yv[i] = y[t * ldy + c];
    }
  };
  fetch(first);
  __syncthreads();
  for (int t0 = first; t0 < last; t0 += kTile) {
    float a[kRunTokens], x[kRunTokens], gy[kRunTokens];
#pragma unroll
    for (int i = 0; i < kRunTokens; ++i) {
      const Step s = make_step<T>(zr[i], zi[i], to_float(uv[i]), b_r, b_i, rt);
      const bool in = t0 + group * kRunTokens + i < last;
      a[i] = in ? s.a : 1.f;  // behind the portion S stays
      x[i] = in ? s.x : 0.f;
      gy[i] = gelu_f<T>(to_float(yv[i]));
    }
    if (t0 + kTile < last) fetch(t0 + kTile);
    const int left = last - t0;
    const int waves = left >= kTile ? kGroups / kQuarters : (left + kRunTokens * kQuarters - 1) / (kRunTokens * kQuarters);
    for (int w = 0; w < waves; ++w) {
      if (w == group / kQuarters) {  // (the whole wavefront)
        float S = carry[threadIdx.x % kChannels];
#pragma unroll
        for (int q = 0; q < kQuarters; ++q) {
          if (q == group % kQuarters) {
#pragma unroll
            for (int i = 0; i < kRunTokens; ++i) {
              S = fmaf(a[i], S, x[i]);
              a[i] = S;
            }
          }
          S = __shfl(S, q * kChannels + threadIdx.x % kChannels, kWave);  // what this quarter ends with, for the next
        }
        if (threadIdx.x % kWave < kChannels) carry[threadIdx.x % kChannels] = S;
      }
      __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < kRunTokens; ++i) {
      const int t = t0 + group * kRunTokens + i;
      if (active && t < last) out[static_cast<size_t>(t) * width + c] = from_float<T>(a[i] * gy[i]);
    }
  }
  if (threadIdx.x < kChannels && active) {
    slot[c] = carry[threadIdx.x];
    keep_tail(slot + width, raw, ld_raw, c, width, taps, first, last, fresh);
  }
}

}  // namespace

}  // namespace shk

using namespace shk;

extern "C" long long shk_rglru_state_floats(int width, int taps) {
  return static_cast<long long>(width) * (taps > 1 ? taps : 1);
}

extern "C" int shk_rglru(const float* gates, int blocks, const float* bias_r, const float* bias_i, const float* rate,
                         const void* u, const void* y, int ldy, const void* raw, int ld_raw, int width, int taps,
                         const int32_t* positions, const int32_t* cu_q, const int32_t* slots, float* state,
                         long long slot_stride, void* out, int dtype, int num_single, int num_seqs, void* stream) {
  SHK_REQUIRE(dtype == kF32 || dtype == kBF16, "rglru: unknown dtype %d", dtype);
  SHK_REQUIRE(width > 0 && blocks > 0 && width % blocks == 0 && taps >= 1 && taps <= 64 && ldy >= width && ld_raw >= width,
              "rglru: bad sizes width=%d blocks=%d taps=%d ldy=%d ld_raw=%d", width, blocks, taps, ldy, ld_raw);
  SHK_REQUIRE(num_single >= 0 && num_seqs >= num_single && num_seqs <= 65535, "rglru: bad number of sequences %d, %d",
              num_single, num_seqs);
  SHK_REQUIRE(slot_stride >= shk_rglru_state_floats(width, taps), "rglru: a slot of %lld floats does not hold the state",
              slot_stride);
  if (num_seqs == 0) return 0;
  SHK_REQUIRE(gates && bias_r && bias_i && rate && u && y && raw && positions && cu_q && slots && state && out,
              "rglru: null pointer");
  hipStream_t s = static_cast<hipStream_t>(stream);
  const int part = width / blocks;
#define SHK_GO(T)                                                                                                     \
  do {                                                                                                                \
    if (num_single > 0)                                                                                               \
      rglru_step_kernel<T><<<dim3((width + 255) / 256, num_single), 256, 0, s>>>(                                     \
          gates, part, bias_r, bias_i, rate, static_cast<const T*>(u), static_cast<const T*>(y), ldy,                 \
          static_cast<const T*>(raw), ld_raw, width, taps, positions, cu_q, slots, state, slot_stride,                \
          static_cast<T*>(out));                                                                                      \
    if (num_seqs > num_single)                                                                                        \
      rglru_scan_kernel<T><<<dim3(blocks_of(width), num_seqs - num_single), 16 * kWave, 0, s>>>(   \
          gates, part, bias_r, bias_i, rate, static_cast<const T*>(u), static_cast<const T*>(y), ldy,                 \
          static_cast<const T*>(raw), ld_raw, width, taps, num_single, positions, cu_q, slots, state, slot_stride,    \
          static_cast<T*>(out));                                                                                      \
  } while (0)
  if (dtype == kF32) SHK_GO(float); else SHK_GO(bf16);
#undef SHK_GO
  SHK_LAUNCH_CHECK("rglru");
  return 0;
}
