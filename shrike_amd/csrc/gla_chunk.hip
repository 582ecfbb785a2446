// Gated linear attention for prompt portions, in chunks on the matrix units:
//   S_t = diag(exp(g_t)) S_(t-1) + k_t v_t^T,   o_t = q_scale S_t^T q_t,
// g [heads, dim] the decays' logarithms (float32, never positive), q, k, v bfloat16 rows.
// Within a chunk of 64 tokens, with c_t the sum of the chunk's g up to t, element by element, and S the
// state before the chunk,
//   o_t = S^T (q_t exp(c_t)) + sum_(s <= t) P[t, s] v_s,   P[t, s] = sum_d q_t k_s exp(c_t - c_s)
//   S  <- diag(exp(c_last)) S + sum_s (k_s exp(c_last - c_s)) v_s^T
// exp(c_t - c_s) with s <= t never exceeds 1, but its two factors exp(c_t) and exp(-c_s) may leave float32's
// range.  So a chunk's scores are formed in blocks of 16 x 16 tokens: between different blocks both factors
// are taken from the sum before the later block (neither exceeds 1), and P is a product of matrices; within
// a block every exponential is formed by itself.
//
// gla_prepare_kernel, a workgroup per (chunk, head), forms what does not depend on the state: P, the decayed
// queries and keys, the chunk's whole decay, laid out as operands of the chain's products (keys and values
// with the tokens innermost).  gla_chain_kernel, a workgroup per (sequence, head, 32 value columns), walks
// the chunks: wavefronts 0 to 3 form the outputs of 16 tokens each, wavefronts 4 to 7 keep the state in their
// registers and form the next one; all operands but the state come straight from memory into registers, a
// chunk ahead, and the state passes through two buffers in LDS: one barrier a chunk.
//
// The state and everything with a decay in it is float32: such an operand of a matrix product enters as the
// sum of two bfloat16 numbers, its rounding and what the rounding left (2^-17 of it is lost); sums are
// float32; the state that goes from chunk to chunk is never rounded.
#include "api.h"
#include "common.h"
#include "mfma_tile.h"

namespace shk {

namespace {

constexpr int kChunk = 64;
constexpr int kVT = 32;  // value columns a workgroup of the chain
constexpr int kVB = kVT / 16;
constexpr int kOutWaves = 4, kChainWaves = 8;
constexpr int kPad = 8;
constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ void split_float(float x, __bf16& hi, __bf16& lo) {
  hi = static_cast<__bf16>(x);
  lo = static_cast<__bf16>(x - static_cast<float>(hi));
}
__device__ __forceinline__ float exp2_f(float x) { return __builtin_amdgcn_exp2f(x); }

// What the two kernels pass on, in one piece of memory (offsets in bytes).
struct Layout {
  size_t q_hi, q_lo;    // [rows][heads][dim]: q exp(c_t) q_scale
  size_t p_hi, p_lo;    // [rows][heads][64]: P, zero for s > t
  size_t k_hi, k_lo;    // [chunks][heads][dim][64]: k exp(c_last - c_s), tokens innermost
  size_t v_t;           // [chunks][heads][v_dim][64]
  size_t decay;         // [chunks][heads][dim] float32: exp(c_last)
  size_t total;
};
__host__ __device__ inline Layout layout_of(size_t rows, size_t chunks, size_t heads, size_t dim, size_t v_dim) {
  Layout l;
  size_t at = 0;
  auto take = [&](size_t bytes) {
    const size_t here = at;
    at += (bytes + 255) / 256 * 256;
    return here;
  };
  l.q_hi = take(rows * heads * dim * 2);
  l.q_lo = take(rows * heads * dim * 2);
  l.p_hi = take(rows * heads * kChunk * 2);
  l.p_lo = take(rows * heads * kChunk * 2);
  l.k_hi = take(chunks * heads * dim * kChunk * 2);
  l.k_lo = take(chunks * heads * dim * kChunk * 2);
  l.v_t = take(chunks * heads * v_dim * kChunk * 2);
  l.decay = take(chunks * heads * dim * 4);
  l.total = at;
  return l;
}

// chunk_seq, chunk_t0 [chunks]: the sequence of a chunk and its first token within the portion
template <int DIM>
__global__ void __launch_bounds__(256)
    gla_prepare_kernel(const bf16* __restrict__ proj, int ld, int q_off, int k_off, int v_off,
                       const float* __restrict__ log_decay, float q_scale, int heads, int v_dim,
                       const int32_t* __restrict__ chunk_seq, const int32_t* __restrict__ chunk_t0,
                       const int32_t* __restrict__ cu_q, char* __restrict__ scratch, Layout at, int first_row) {
  constexpr int BS = DIM + 4;     // float32 between rows of the sums (16-byte rows)
  constexpr int KS = DIM + kPad;  // bfloat16 between rows of queries and keys
  constexpr int DS = DIM / 32;
  __shared__ __attribute__((aligned(16))) float sums[kChunk][BS];  // c_t / ln 2
  __shared__ __attribute__((aligned(16))) __bf16 qs[kChunk][KS], ks[kChunk][KS];
  const int h = blockIdx.x, chunk = blockIdx.y;
  const int seq = chunk_seq[chunk], t0 = chunk_t0[chunk];
  const int first = cu_q[seq] + t0, len = cu_q[seq + 1] - first;
  if (len <= 0) return;
  const int count = len < kChunk ? len : kChunk;
  const int tid = threadIdx.x, wave = tid / kWave, lane = tid % kWave, j = lane % 16, g = lane / 16;

  for (int i = tid; i < kChunk * DIM / 8; i += 256) {
    const int t = i / (DIM / 8), d = i % (DIM / 8) * 8;
    uint4 q = make_uint4(0, 0, 0, 0), k = make_uint4(0, 0, 0, 0);
    if (t < count) {
      const bf16* row = proj + static_cast<size_t>(first + t) * ld + h * DIM + d;
      q = *reinterpret_cast<const uint4*>(row + q_off);
      k = *reinterpret_cast<const uint4*>(row + k_off);
    }
    *reinterpret_cast<uint4*>(&qs[t][d]) = q;
    *reinterpret_cast<uint4*>(&ks[t][d]) = k;
  }
  for (int i = tid; i < kChunk * DIM / 4; i += 256) {
    const int t = i / (DIM / 4), d = i % (DIM / 4) * 4;
    float4 x = make_float4(0.f, 0.f, 0.f, 0.f);  // behind the portion nothing decays
    if (t < count) x = *reinterpret_cast<const float4*>(log_decay + (static_cast<size_t>(first + t) * heads + h) * DIM + d);
    *reinterpret_cast<float4*>(&sums[t][d]) = make_float4(x.x * kLog2e, x.y * kLog2e, x.z * kLog2e, x.w * kLog2e);
  }
  __syncthreads();
  if (tid < DIM) {
    float run = 0.f;
#pragma unroll 16
    for (int t = 0; t < kChunk; ++t) {
      run += sums[t][tid];
      sums[t][tid] = run;
    }
    reinterpret_cast<float*>(scratch + at.decay)[(static_cast<size_t>(chunk) * heads + h) * DIM + tid] = exp2_f(run);
  }
  __syncthreads();

  // decayed queries, row by row
  __bf16* q_hi = reinterpret_cast<__bf16*>(scratch + at.q_hi);
  __bf16* q_lo = reinterpret_cast<__bf16*>(scratch + at.q_lo);
  for (int i = tid; i < count * (DIM / 8); i += 256) {
    const int t = i / (DIM / 8), d = i % (DIM / 8) * 8;
    AFrag hi, lo;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      __bf16 a, b;
      split_float(static_cast<float>(qs[t][d + e]) * q_scale * exp2_f(sums[t][d + e]), a, b);
      hi.v[e] = a, lo.v[e] = b;
    }
    const size_t dst = (static_cast<size_t>(first - first_row + t) * heads + h) * DIM + d;
    *reinterpret_cast<uint4*>(q_hi + dst) = hi.u;
    *reinterpret_cast<uint4*>(q_lo + dst) = lo.u;
  }
  // decayed keys and the values, eight tokens of an element side by side
  __bf16* k_hi = reinterpret_cast<__bf16*>(scratch + at.k_hi) + (static_cast<size_t>(chunk) * heads + h) * DIM * kChunk;
  __bf16* k_lo = reinterpret_cast<__bf16*>(scratch + at.k_lo) + (static_cast<size_t>(chunk) * heads + h) * DIM * kChunk;
  for (int i = tid; i < DIM * (kChunk / 8); i += 256) {
    const int s = i % (kChunk / 8) * 8, d = i / (kChunk / 8);
    const float end = sums[kChunk - 1][d];
    AFrag hi, lo;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      __bf16 a, b;
      split_float(static_cast<float>(ks[s + e][d]) * exp2_f(end - sums[s + e][d]), a, b);
      hi.v[e] = a, lo.v[e] = b;
    }
    *reinterpret_cast<uint4*>(k_hi + static_cast<size_t>(d) * kChunk + s) = hi.u;
    *reinterpret_cast<uint4*>(k_lo + static_cast<size_t>(d) * kChunk + s) = lo.u;
  }
  uint16_t* v_t = reinterpret_cast<uint16_t*>(scratch + at.v_t) + (static_cast<size_t>(chunk) * heads + h) * v_dim * kChunk;
  for (int i = tid; i < v_dim * (kChunk / 8); i += 256) {
    const int c = i % v_dim, s = i / v_dim * 8;
    AFrag x;
#pragma unroll
    for (int e = 0; e < 8; ++e)
      x.h[e] = s + e < count ? proj[static_cast<size_t>(first + s + e) * ld + v_off + h * v_dim + c].bits : 0;
    *reinterpret_cast<uint4*>(v_t + static_cast<size_t>(c) * kChunk + s) = x.u;
  }

  // scores: wavefront w forms rows 16 w .. 16 w + 15
  __bf16* p_hi = reinterpret_cast<__bf16*>(scratch + at.p_hi);
  __bf16* p_lo = reinterpret_cast<__bf16*>(scratch + at.p_lo);
  const int r0 = 16 * wave, t = r0 + j;
  const size_t prow = (static_cast<size_t>(first - first_row + t) * heads + h) * kChunk;
  auto put = [&](int s, const float (&x)[4]) {  // P[t][s .. s + 3]
    if (t >= count) return;
    uint2 hi, lo;
    __bf16 a[4], b[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) split_float(x[r], a[r], b[r]);
    hi.x = __builtin_bit_cast(uint16_t, a[0]) | (static_cast<uint32_t>(__builtin_bit_cast(uint16_t, a[1])) << 16);
    hi.y = __builtin_bit_cast(uint16_t, a[2]) | (static_cast<uint32_t>(__builtin_bit_cast(uint16_t, a[3])) << 16);
    lo.x = __builtin_bit_cast(uint16_t, b[0]) | (static_cast<uint32_t>(__builtin_bit_cast(uint16_t, b[1])) << 16);
    lo.y = __builtin_bit_cast(uint16_t, b[2]) | (static_cast<uint32_t>(__builtin_bit_cast(uint16_t, b[3])) << 16);
    *reinterpret_cast<uint2*>(p_hi + prow + s) = hi;
    *reinterpret_cast<uint2*>(p_lo + prow + s) = lo;
  };
  if (r0 < count) {
    if (wave > 0) {
      f32x4 acc[3];
#pragma unroll
      for (int b = 0; b < 3; ++b) acc[b] = f32x4{0.f, 0.f, 0.f, 0.f};
      for (int ds = 0; ds < DS; ++ds) {
        const int d = ds * 32 + g * 8;
        float base[8];
        AFrag qh, ql;
#pragma unroll
        for (int e = 0; e < 8; ++e) base[e] = sums[r0 - 1][d + e];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          __bf16 a, b;
          split_float(static_cast<float>(qs[t][d + e]) * q_scale * exp2_f(sums[t][d + e] - base[e]), a, b);
          qh.v[e] = a, ql.v[e] = b;
        }
#pragma unroll
        for (int b = 0; b < 3; ++b) {
          if (b >= wave) break;
          AFrag kh, kl;
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            __bf16 x, y;
            split_float(static_cast<float>(ks[16 * b + j][d + e]) * exp2_f(base[e] - sums[16 * b + j][d + e]), x, y);
            kh.v[e] = x, kl.v[e] = y;
          }
          acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh.v, qh.v, acc[b], 0, 0, 0);
          acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kl.v, qh.v, acc[b], 0, 0, 0);
          acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh.v, ql.v, acc[b], 0, 0, 0);
        }
      }
#pragma unroll
      for (int b = 0; b < 3; ++b) {
        if (b >= wave) break;
        const float x[4] = {acc[b][0], acc[b][1], acc[b][2], acc[b][3]};
        put(16 * b + 4 * g, x);
      }
    }
    // within the block: this lane takes token t and the keys r0 + 4 g .. + 3
    float x[4] = {0.f, 0.f, 0.f, 0.f};
    for (int d = 0; d < DIM; d += 4) {
      const float4 ct = *reinterpret_cast<const float4*>(&sums[t][d]);
      const float c[4] = {ct.x, ct.y, ct.z, ct.w};
      float q[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) q[e] = static_cast<float>(qs[t][d + e]);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int s = r0 + 4 * g + r;
        const float4 cs = *reinterpret_cast<const float4*>(&sums[s][d]);
        const float c2[4] = {cs.x, cs.y, cs.z, cs.w};
#pragma unroll
        for (int e = 0; e < 4; ++e)
          x[r] = fmaf(q[e] * static_cast<float>(ks[s][d + e]), exp2_f(c[e] - c2[e]), x[r]);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) x[r] = r0 + 4 * g + r <= t ? x[r] * q_scale : 0.f;
    put(r0 + 4 * g, x);
    const float zero[4] = {0.f, 0.f, 0.f, 0.f};
    for (int b = wave + 1; b < kChunk / 16; ++b) put(16 * b + 4 * g, zero);
  }
}

// chunk_base[i]: the first chunk of portion i (sequence first_seq + i)
template <int DIM>
__global__ void __launch_bounds__(kChainWaves* kWave)
    gla_chain_kernel(const char* __restrict__ scratch, Layout at, int first_row, int heads, int v_dim, int first_seq,
                     const int32_t* __restrict__ chunk_base, const int32_t* __restrict__ positions,
                     const int32_t* __restrict__ cu_q, const int32_t* __restrict__ slots, float* __restrict__ state,
                     long long slot_stride, float* __restrict__ out) {
  constexpr int DS = DIM / 32;
  constexpr int NT = (DIM / 16 + kOutWaves - 1) / kOutWaves;  // blocks of the state a wavefront owns
  __shared__ __attribute__((aligned(16))) __bf16 s_hi[2][kVT][DIM + kPad], s_lo[2][kVT][DIM + kPad];
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, j = lane % 16, g = lane / 16;
  const bool outputs = wave < kOutWaves;
  const int own = wave % kOutWaves;  // tokens 16 own .. + 15, or the state's blocks own, own + 4, ...
  const int tiles = v_dim / kVT;
  const int h = blockIdx.x / tiles, v0 = blockIdx.x % tiles * kVT;
  const int seq = first_seq + blockIdx.y;
  const int first = cu_q[seq], len = cu_q[seq + 1] - first;
  if (len <= 0) return;
  const int base = chunk_base[blockIdx.y];
  const bool fresh = positions[first] == 0;
  float* srow = state + static_cast<size_t>(slots[seq]) * slot_stride + (static_cast<size_t>(h) * v_dim + v0) * DIM;
  const __bf16* q_hi = reinterpret_cast<const __bf16*>(scratch + at.q_hi);
  const __bf16* q_lo = reinterpret_cast<const __bf16*>(scratch + at.q_lo);
  const __bf16* p_hi = reinterpret_cast<const __bf16*>(scratch + at.p_hi);
  const __bf16* p_lo = reinterpret_cast<const __bf16*>(scratch + at.p_lo);
  const __bf16* k_hi = reinterpret_cast<const __bf16*>(scratch + at.k_hi);
  const __bf16* k_lo = reinterpret_cast<const __bf16*>(scratch + at.k_lo);
  const __bf16* v_t = reinterpret_cast<const __bf16*>(scratch + at.v_t);
  const float* decay = reinterpret_cast<const float*>(scratch + at.decay);
  auto load = [](const __bf16* p) {
    AFrag f;
    f.u = *reinterpret_cast<const uint4*>(p);
    return f;
  };
  const int chunks = (len + kChunk - 1) / kChunk;

  if (outputs) {
    AFrag qh[DS], ql[DS], ph[2], pl[2], vf[kVB][2];
    auto fetch = [&](int c) {  // (tokens behind the portion read its last one; their outputs are dropped)
      const int tt = c * kChunk + 16 * own + j;
      const size_t row = static_cast<size_t>(first - first_row + (tt < len ? tt : len - 1)) * heads + h;
#pragma unroll
      for (int ds = 0; ds < DS; ++ds) {
        qh[ds] = load(q_hi + row * DIM + ds * 32 + g * 8);
        ql[ds] = load(q_lo + row * DIM + ds * 32 + g * 8);
      }
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        ph[s] = load(p_hi + row * kChunk + s * 32 + g * 8);
        pl[s] = load(p_lo + row * kChunk + s * 32 + g * 8);
#pragma unroll
        for (int vb = 0; vb < kVB; ++vb)
          vf[vb][s] = load(v_t + ((static_cast<size_t>(base + c) * heads + h) * v_dim + v0 + 16 * vb + j) * kChunk + s * 32 + g * 8);
      }
    };
    fetch(0);
    for (int c = 0; c < chunks; ++c) {
      AFrag ch[DS], cl[DS], cph[2], cpl[2], cvf[kVB][2];
#pragma unroll
      for (int ds = 0; ds < DS; ++ds) ch[ds] = qh[ds], cl[ds] = ql[ds];
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        cph[s] = ph[s], cpl[s] = pl[s];
#pragma unroll
        for (int vb = 0; vb < kVB; ++vb) cvf[vb][s] = vf[vb][s];
      }
      if (c + 1 < chunks) fetch(c + 1);
      // what the state does not enter first: O^T = V^T P^T
      f32x4 o[kVB];
#pragma unroll
      for (int vb = 0; vb < kVB; ++vb) {
        o[vb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < 2; ++s) {
          o[vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cvf[vb][s].v, cph[s].v, o[vb], 0, 0, 0);
          o[vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cvf[vb][s].v, cpl[s].v, o[vb], 0, 0, 0);
        }
      }
      __syncthreads();  // the state before this chunk is in buffer c % 2
#pragma unroll
      for (int ds = 0; ds < DS; ++ds)
#pragma unroll
        for (int vb = 0; vb < kVB; ++vb) {
          const AFrag hi = load(&s_hi[c % 2][16 * vb + j][ds * 32 + g * 8]);
          const AFrag lo = load(&s_lo[c % 2][16 * vb + j][ds * 32 + g * 8]);
          o[vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi.v, ch[ds].v, o[vb], 0, 0, 0);
          o[vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo.v, ch[ds].v, o[vb], 0, 0, 0);
          o[vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi.v, cl[ds].v, o[vb], 0, 0, 0);
        }
      const int tt = c * kChunk + 16 * own + j;
      if (tt < len) {
        float* dst = out + (static_cast<size_t>(first + tt) * heads + h) * v_dim + v0 + 4 * g;
#pragma unroll
        for (int vb = 0; vb < kVB; ++vb)
          *reinterpret_cast<float4*>(dst + 16 * vb) = make_float4(o[vb][0], o[vb][1], o[vb][2], o[vb][3]);
      }
    }
    return;
  }

  // the state: block b = own + 4 nt of 16 elements d = 16 b + j, columns v = 16 vb + 4 g + r
  f32x4 S[NT][kVB];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt)
#pragma unroll
    for (int vb = 0; vb < kVB; ++vb) {
      const int d = (own + kOutWaves * nt) * 16 + j;
      S[nt][vb] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (!fresh && d < DIM) {
#pragma unroll
        for (int r = 0; r < 4; ++r) S[nt][vb][r] = srow[static_cast<size_t>(16 * vb + 4 * g + r) * DIM + d];
      }
    }
  AFrag kh[NT][2], kl[NT][2], vf[kVB][2];
  float whole[NT];
  auto fetch = [&](int c) {
    const size_t ch = static_cast<size_t>(base + c) * heads + h;
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      const int b = own + kOutWaves * nt;
      const int d = (b * 16 < DIM ? b * 16 : 0) + j;
      whole[nt] = decay[ch * DIM + d];
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        kh[nt][s] = load(k_hi + (ch * DIM + d) * kChunk + s * 32 + g * 8);
        kl[nt][s] = load(k_lo + (ch * DIM + d) * kChunk + s * 32 + g * 8);
      }
    }
#pragma unroll
    for (int vb = 0; vb < kVB; ++vb)
#pragma unroll
      for (int s = 0; s < 2; ++s) vf[vb][s] = load(v_t + (ch * v_dim + v0 + 16 * vb + j) * kChunk + s * 32 + g * 8);
  };
  fetch(0);
  for (int c = 0; c < chunks; ++c) {
    // this chunk's operands aside, so that the next one's are on their way while the state is published and multiplied
    AFrag ckh[NT][2], ckl[NT][2], cvf[kVB][2];
    float cwhole[NT];
#pragma unroll
    for (int s = 0; s < 2; ++s) {
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) ckh[nt][s] = kh[nt][s], ckl[nt][s] = kl[nt][s];
#pragma unroll
      for (int vb = 0; vb < kVB; ++vb) cvf[vb][s] = vf[vb][s];
    }
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) cwhole[nt] = whole[nt];
    if (c + 1 < chunks) fetch(c + 1);
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      const int d = (own + kOutWaves * nt) * 16 + j;
      if (d >= DIM) break;
#pragma unroll
      for (int vb = 0; vb < kVB; ++vb)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          split_float(S[nt][vb][r], s_hi[c % 2][16 * vb + 4 * g + r][d], s_lo[c % 2][16 * vb + 4 * g + r][d]);
    }
    __syncthreads();
#pragma unroll
    for (int nt = 0; nt < NT; ++nt)
#pragma unroll
      for (int vb = 0; vb < kVB; ++vb) {
        S[nt][vb] *= cwhole[nt];
#pragma unroll
        for (int s = 0; s < 2; ++s) {
          S[nt][vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cvf[vb][s].v, ckh[nt][s].v, S[nt][vb], 0, 0, 0);
          S[nt][vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cvf[vb][s].v, ckl[nt][s].v, S[nt][vb], 0, 0, 0);
        }
      }
  }
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) {
    const int d = (own + kOutWaves * nt) * 16 + j;
    if (d >= DIM) break;
#pragma unroll
    for (int vb = 0; vb < kVB; ++vb)
#pragma unroll
      for (int r = 0; r < 4; ++r) srow[static_cast<size_t>(16 * vb + 4 * g + r) * DIM + d] = S[nt][vb][r];
  }
}

}  // namespace

}  // namespace shk

using namespace shk;

extern "C" int shk_gla_chunk_supports(int dim, int v_dim) {
  const bool size = dim == 32 || dim == 64 || dim == 96 || dim == 128 || dim == 192 || dim == 256;
  return size && v_dim > 0 && v_dim % kVT == 0;
}

extern "C" long long shk_gla_chunk_scratch_bytes(int rows, int chunks, int heads, int dim, int v_dim) {
  return static_cast<long long>(layout_of(rows, chunks, heads, dim, v_dim).total);
}

extern "C" int shk_gla_chunk_bf16(const void* proj, int ld, int q_off, int k_off, int v_off, const float* log_decay,
                                  float q_scale, int first_seq, int num_seqs, int first_row, int rows, int heads, int dim,
                                  int v_dim, const int32_t* chunk_lists, int chunks, const int32_t* positions,
                                  const int32_t* cu_q, const int32_t* slots, float* state, long long slot_stride,
                                  void* scratch, float* out, void* stream) {
  SHK_REQUIRE(first_seq >= 0 && num_seqs >= 0 && first_row >= 0 && rows >= 0 && chunks >= 0 && heads > 0 &&
                  shk_gla_chunk_supports(dim, v_dim),
              "gla_chunk: bad sizes seqs=%d heads=%d dim=%d v_dim=%d", num_seqs, heads, dim, v_dim);
  SHK_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && q_off + heads * dim <= ld && k_off + heads * dim <= ld &&
                  v_off + heads * v_dim <= ld && q_off % 8 == 0 && k_off % 8 == 0 && ld % 8 == 0,
              "gla_chunk: columns do not fit rows of %d, or are not in runs of 8", ld);
  SHK_REQUIRE(slot_stride >= shk_retention_state_floats(heads, dim, v_dim),
              "gla_chunk: a slot of %lld floats does not hold the state", slot_stride);
  if (num_seqs == 0 || rows == 0) return 0;
  SHK_REQUIRE(num_seqs <= 65535 && chunks <= 65535 && chunks >= num_seqs, "gla_chunk: %d sequences in %d chunks", num_seqs,
              chunks);
  SHK_REQUIRE(proj && log_decay && chunk_lists && positions && cu_q && slots && state && scratch && out,
              "gla_chunk: null pointer");
  SHK_REQUIRE(reinterpret_cast<uintptr_t>(proj) % 16 == 0 && reinterpret_cast<uintptr_t>(out) % 16 == 0 &&
                  reinterpret_cast<uintptr_t>(log_decay) % 16 == 0 && reinterpret_cast<uintptr_t>(scratch) % 16 == 0,
              "gla_chunk: proj, log_decay, scratch and out must be 16-byte aligned");
  hipStream_t s = static_cast<hipStream_t>(stream);
  const Layout at = layout_of(rows, chunks, heads, dim, v_dim);
#define SHK_GO(D)                                                                                                       \
  do {                                                                                                                  \
    gla_prepare_kernel<D><<<dim3(heads, chunks), 256, 0, s>>>(static_cast<const bf16*>(proj), ld, q_off, k_off, v_off,  \
                                                              log_decay, q_scale, heads, v_dim, chunk_lists,            \
                                                              chunk_lists + chunks, cu_q, static_cast<char*>(scratch), at, \
                                                              first_row);                                               \
    gla_chain_kernel<D><<<dim3(heads * (v_dim / kVT), num_seqs), kChainWaves * kWave, 0, s>>>(                          \
        static_cast<const char*>(scratch), at, first_row, heads, v_dim, first_seq, chunk_lists + 2 * chunks, positions, \
        cu_q, slots, state, slot_stride, out);                                                                          \
  } while (0)
  switch (dim) {
    case 32: SHK_GO(32); break;
    case 64: SHK_GO(64); break;
    case 96: SHK_GO(96); break;
    case 128: SHK_GO(128); break;
    case 192: SHK_GO(192); break;
    default: SHK_GO(256); break;
  }
#undef SHK_GO
  SHK_LAUNCH_CHECK("gla_chunk");
  return 0;
}
