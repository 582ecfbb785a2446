// Linear attention with a fixed decay per head for prompt portions, in chunks on the matrix units:
//   S_t = decay S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,   q, k, v bfloat16 rows.
// Within a chunk of 64 tokens, with a = decay and S the state before it,
//   o_t = a^(t+1) S^T q_t + sum_(s <= t) a^(t-s) (q_t . k_s) v_s
//   S  <- a^n S + sum_s a^(n-1-s) k_s v_s^T
// so a chunk is four products of matrices, and the chain from token to token is a chain from chunk to
// chunk.  The state and everything with a decay in it is float32: a float32 operand of a matrix product
// (decayed scores, decayed values, the state) enters as the sum of two bfloat16 numbers, its rounding
// and what the rounding left (two matrix instructions; what is lost is 2^-17 of the operand); sums are
// float32; the state that goes from chunk to chunk is never rounded.
//
// A workgroup of eight wavefronts owns (sequence, head, 32 value columns).  Everything is formed
// transposed.  Wavefronts 0 to 3 form the chunk's outputs, wavefront w those of the tokens 16 w .. 16 w +
// 15 as columns: P^T = K Q^T comes out as the operand that O^T += V^T P^T takes (keys assigned to the first
// product's rows so that a lane ends up with 8 consecutive ones), O^T starts as S^T Q^T.  Wavefronts 4 to
// 7 meanwhile form the next state, S^T += V^T K, every fourth block of 16 elements of the keys' size
// each, whose float32 sums stay in their registers from chunk to chunk.  A wavefront issues an instruction
// every four to five cycles whatever its kind, so the chain is as long as the instructions of one
// wavefront: hence the two roles, and everything that all wavefronts need formed once while a chunk is
// staged.  In LDS: keys both ways round, values transposed, the decayed values' and the state's two halves;
// the next chunk's rows are on their way into registers while a chunk is multiplied.
#include "api.h"
#include "common.h"
#include "mfma_tile.h"

namespace shk {

namespace {

constexpr int kChunk = 64;
constexpr int kVT = 32;       // value columns a workgroup
constexpr int kOutWaves = 4, kChunkWaves = 8;
constexpr int kPad = 8;       // bfloat16 elements behind an LDS row, so that operand reads meet every bank

// x as the sum of two bfloat16 numbers
__device__ __forceinline__ void split_float(float x, __bf16& hi, __bf16& lo) {
  hi = static_cast<__bf16>(x);
  lo = static_cast<__bf16>(x - static_cast<float>(hi));
}

template <int DIM>
__global__ void __launch_bounds__(kChunkWaves* kWave)
    retention_chunk_kernel(const bf16* __restrict__ proj, int ld, int q_off, int k_off, int v_off,
                           const float* __restrict__ decay, int heads, int v_dim, int first_seq,
                           const int32_t* __restrict__ positions, const int32_t* __restrict__ cu_q,
                           const int32_t* __restrict__ slots, float* __restrict__ state, long long slot_stride,
                           float* __restrict__ out) {
  constexpr int DS = DIM / 32;                                    // operand slices of a query or key
  constexpr int NT = (DIM / 16 + kOutWaves - 1) / kOutWaves;      // blocks of the state a wavefront owns
  constexpr int KR = (DIM / 8 + kChunkWaves - 1) / kChunkWaves;   // runs of 8 key elements a thread stages
  constexpr int VB = kVT / 16;
  __shared__ __attribute__((aligned(16))) __bf16 keys[kChunk][DIM + kPad];     // [token][element]
  __shared__ __attribute__((aligned(16))) __bf16 keys_t[DIM][kChunk + kPad];   // [element][token]
  __shared__ __attribute__((aligned(16))) __bf16 values_t[kVT][kChunk + kPad]; // [column][token]
  __shared__ __attribute__((aligned(16))) __bf16 v_hi[kVT][kChunk + kPad], v_lo[kVT][kChunk + kPad];  // decayed
  __shared__ __attribute__((aligned(16))) __bf16 s_hi[kVT][DIM + kPad], s_lo[kVT][DIM + kPad];
  __shared__ float pw[kChunk + 1];  // decay^i

  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, j = lane % 16, g = lane / 16;
  const bool outputs = wave < kOutWaves;
  const int own = wave % kOutWaves;  // tokens 16 own .. + 15, or the state's blocks own, own + 4, ...
  const int tiles = v_dim / kVT;
  const int h = blockIdx.x / tiles, v0 = blockIdx.x % tiles * kVT;
  const int seq = first_seq + blockIdx.y;
  const int first = cu_q[seq], len = cu_q[seq + 1] - first;
  if (len <= 0) return;
  const bool fresh = positions[first] == 0;
  float* srow = state + static_cast<size_t>(slots[seq]) * slot_stride + (static_cast<size_t>(h) * v_dim + v0) * DIM;
  if (threadIdx.x <= kChunk) pw[threadIdx.x] = threadIdx.x == 0 ? 1.f : powf(decay[h], static_cast<float>(threadIdx.x));

  // the state: block b = own + 4 nt of 16 elements d = 16 b + j, columns v = 16 vb + 4 g + r
  f32x4 S[NT][VB];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt)
#pragma unroll
    for (int vb = 0; vb < VB; ++vb) {
      const int d = (own + kOutWaves * nt) * 16 + j;
      S[nt][vb] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (!fresh && !outputs && d < DIM) {
#pragma unroll
        for (int r = 0; r < 4; ++r) S[nt][vb][r] = srow[static_cast<size_t>(16 * vb + 4 * g + r) * DIM + d];
      }
    }

  AFrag raw_k[KR], raw_v, raw_q[DS];
  // Every load is unconditional: tokens behind the portion read its last one.  A lane stages its own token
  // (lane = token of the chunk) of keys and values; queries are operands as they lie.
  auto fetch = [&](int t0) {
    const int tk = t0 + lane < len ? t0 + lane : len - 1;
    const bf16* row = proj + static_cast<size_t>(first + tk) * ld;
#pragma unroll
    for (int i = 0; i < KR; ++i) {
      const int run = wave * KR + i < DIM / 8 ? wave * KR + i : DIM / 8 - 1;
      raw_k[i].u = *reinterpret_cast<const uint4*>(row + k_off + h * DIM + run * 8);
    }
    raw_v.u = *reinterpret_cast<const uint4*>(row + v_off + h * v_dim + v0 + own * 8);
    const int tq = t0 + 16 * own + j < len ? t0 + 16 * own + j : len - 1;
    const bf16* qrow = proj + static_cast<size_t>(first + tq) * ld + q_off + h * DIM + g * 8;
#pragma unroll
    for (int ds = 0; ds < DS; ++ds) raw_q[ds].u = *reinterpret_cast<const uint4*>(qrow + ds * 32);
  };
  AFrag qf[DS];
  auto stage = [&](int count) {  // what was fetched, into LDS and the query operands
    const bool in = lane < count;  // tokens behind the chunk's end are zero rows
#pragma unroll
    for (int i = 0; i < KR; ++i) {
      const int run = wave * KR + i;
      if (run >= DIM / 8) break;
      AFrag x = raw_k[i];
      if (!in) x.u = make_uint4(0, 0, 0, 0);
      *reinterpret_cast<uint4*>(&keys[lane][run * 8]) = x.u;
#pragma unroll
      for (int e = 0; e < 8; ++e) keys_t[run * 8 + e][lane] = x.v[e];
    }
    AFrag x = raw_v;
    if (!in) x.u = make_uint4(0, 0, 0, 0);
    if (outputs) {
#pragma unroll
      for (int e = 0; e < 8; ++e) values_t[own * 8 + e][lane] = x.v[e];
#pragma unroll
      for (int ds = 0; ds < DS; ++ds) qf[ds] = raw_q[ds];
    } else {
      const float decayed = in ? pw[count - 1 - lane] : 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e)
        split_float(static_cast<float>(x.v[e]) * decayed, v_hi[own * 8 + e][lane], v_lo[own * 8 + e][lane]);
    }
  };
  auto publish = [&]() {  // the state, as two bfloat16 numbers, for S^T Q^T
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      const int d = (own + kOutWaves * nt) * 16 + j;
      if (d >= DIM) break;
#pragma unroll
      for (int vb = 0; vb < VB; ++vb)
#pragma unroll
        for (int r = 0; r < 4; ++r) split_float(S[nt][vb][r], s_hi[16 * vb + 4 * g + r][d], s_lo[16 * vb + 4 * g + r][d]);
    }
  };

  fetch(0);
  __syncthreads();  // the powers of the decay
  stage(len < kChunk ? len : kChunk);
  if (!outputs) publish();
  for (int t0 = 0; t0 < len; t0 += kChunk) {
    const int count = len - t0 < kChunk ? len - t0 : kChunk;
    __syncthreads();
    const bool more = t0 + kChunk < len;
    fetch(more ? t0 + kChunk : t0);
    if (outputs) {
      // O^T = S^T Q^T a^(t+1) + V^T P^T for this wavefront's tokens (column j: token t)
      const int t = 16 * own + j;
      f32x4 o[VB];
#pragma unroll
      for (int vb = 0; vb < VB; ++vb) o[vb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ds = 0; ds < DS; ++ds)
#pragma unroll
        for (int vb = 0; vb < VB; ++vb) {
          AFrag hi, lo;
          hi.u = *reinterpret_cast<const uint4*>(&s_hi[16 * vb + j][ds * 32 + g * 8]);
          lo.u = *reinterpret_cast<const uint4*>(&s_lo[16 * vb + j][ds * 32 + g * 8]);
          o[vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi.v, qf[ds].v, o[vb], 0, 0, 0);
          o[vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo.v, qf[ds].v, o[vb], 0, 0, 0);
        }
#pragma unroll
      for (int vb = 0; vb < VB; ++vb) o[vb] *= pw[t + 1];
      for (int s0 = 0; s0 <= 16 * own + 15; s0 += 32) {  // 32 keys at a time, none after the last token
        f32x4 sc[2];
        sc[0] = sc[1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ds = 0; ds < DS; ++ds)
#pragma unroll
          for (int tt = 0; tt < 2; ++tt) {
            AFrag kf;
            kf.u = *reinterpret_cast<const uint4*>(&keys[s0 + 8 * (j / 4) + 4 * tt + j % 4][ds * 32 + g * 8]);
            sc[tt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf.v, qf[ds].v, sc[tt], 0, 0, 0);
          }
        AFrag hi, lo;  // keys s0 + 8 g + e of this lane's token
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int back = t - (s0 + 8 * g + e);
          const float p = pw[back > 0 ? back : 0];
          __bf16 a, b;
          split_float(back >= 0 ? sc[e / 4][e % 4] * p : 0.f, a, b);
          hi.v[e] = a, lo.v[e] = b;
        }
#pragma unroll
        for (int vb = 0; vb < VB; ++vb) {
          AFrag vf;
          vf.u = *reinterpret_cast<const uint4*>(&values_t[16 * vb + j][s0 + g * 8]);
          o[vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf.v, hi.v, o[vb], 0, 0, 0);
          o[vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf.v, lo.v, o[vb], 0, 0, 0);
        }
      }
      if (t < count) {
        float* dst = out + (static_cast<size_t>(first + t0 + t) * heads + h) * v_dim + v0 + 4 * g;
#pragma unroll
        for (int vb = 0; vb < VB; ++vb)
          *reinterpret_cast<float4*>(dst + 16 * vb) = make_float4(o[vb][0], o[vb][1], o[vb][2], o[vb][3]);
      }
    } else {
      // S^T <- a^n S^T + (V^T with column s times a^(n-1-s)) K
      const float whole = pw[count];
#pragma unroll
      for (int nt = 0; nt < NT; ++nt)
#pragma unroll
        for (int vb = 0; vb < VB; ++vb) S[nt][vb] *= whole;
#pragma unroll
      for (int s0 = 0; s0 < kChunk; s0 += 32) {
        AFrag hi[VB], lo[VB];
#pragma unroll
        for (int vb = 0; vb < VB; ++vb) {
          hi[vb].u = *reinterpret_cast<const uint4*>(&v_hi[16 * vb + j][s0 + g * 8]);
          lo[vb].u = *reinterpret_cast<const uint4*>(&v_lo[16 * vb + j][s0 + g * 8]);
        }
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
          const int b = own + kOutWaves * nt;
          if (b * 16 >= DIM) break;
          AFrag kf;
          kf.u = *reinterpret_cast<const uint4*>(&keys_t[b * 16 + j][s0 + g * 8]);
#pragma unroll
          for (int vb = 0; vb < VB; ++vb) {
            S[nt][vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi[vb].v, kf.v, S[nt][vb], 0, 0, 0);
            S[nt][vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo[vb].v, kf.v, S[nt][vb], 0, 0, 0);
          }
        }
      }
    }
    __syncthreads();  // the chunk's operands are read no more
    if (more) {
      stage(len - t0 - kChunk < kChunk ? len - t0 - kChunk : kChunk);
      if (!outputs) publish();
    }
  }
  if (outputs) return;
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) {
    const int d = (own + kOutWaves * nt) * 16 + j;
    if (d >= DIM) break;
#pragma unroll
    for (int vb = 0; vb < VB; ++vb)
#pragma unroll
      for (int r = 0; r < 4; ++r) srow[static_cast<size_t>(16 * vb + 4 * g + r) * DIM + d] = S[nt][vb][r];
  }
}

}  // namespace

}  // namespace shk

using namespace shk;

extern "C" int shk_retention_chunk_supports(int dim, int v_dim) {
  const bool size = dim == 32 || dim == 64 || dim == 96 || dim == 128 || dim == 192 || dim == 256;
  return size && v_dim > 0 && v_dim % kVT == 0;
}

extern "C" int shk_retention_chunk_bf16(const void* proj, int ld, int q_off, int k_off, int v_off, const float* decay,
                                        int first_seq, int num_seqs, int heads, int dim, int v_dim,
                                        const int32_t* positions, const int32_t* cu_q, const int32_t* slots, float* state,
                                        long long slot_stride, float* out, void* stream) {
  SHK_REQUIRE(first_seq >= 0 && num_seqs >= 0 && heads > 0 && shk_retention_chunk_supports(dim, v_dim),
              "retention_chunk: bad sizes seqs=%d heads=%d dim=%d v_dim=%d", num_seqs, heads, dim, v_dim);
  SHK_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && q_off + heads * dim <= ld && k_off + heads * dim <= ld &&
                  v_off + heads * v_dim <= ld && q_off % 8 == 0 && k_off % 8 == 0 && v_off % 8 == 0 && ld % 8 == 0,
              "retention_chunk: columns do not fit rows of %d, or are not in runs of 8", ld);
  SHK_REQUIRE(slot_stride >= shk_retention_state_floats(heads, dim, v_dim),
              "retention_chunk: a slot of %lld floats does not hold the state", slot_stride);
  if (num_seqs == 0) return 0;
  SHK_REQUIRE(num_seqs <= 65535, "retention_chunk: at most 65535 sequences a call");
  SHK_REQUIRE(proj && decay && positions && cu_q && slots && state && out, "retention_chunk: null pointer");
  SHK_REQUIRE(reinterpret_cast<uintptr_t>(proj) % 16 == 0 && reinterpret_cast<uintptr_t>(out) % 16 == 0,
              "retention_chunk: proj and out must be 16-byte aligned");
  hipStream_t s = static_cast<hipStream_t>(stream);
  const dim3 grid(heads * (v_dim / kVT), num_seqs);
#define SHK_GO(D)                                                                                              \
  retention_chunk_kernel<D><<<grid, kChunkWaves * kWave, 0, s>>>(static_cast<const bf16*>(proj), ld, q_off, k_off, \
                                                                 v_off, decay, heads, v_dim, first_seq, positions, \
                                                                 cu_q, slots, state, slot_stride, out)
  switch (dim) {
    case 32: SHK_GO(32); break;
    case 64: SHK_GO(64); break;
    case 96: SHK_GO(96); break;
    case 128: SHK_GO(128); break;
    case 192: SHK_GO(192); break;
    default: SHK_GO(256); break;
  }
#undef SHK_GO
  SHK_LAUNCH_CHECK("retention_chunk");
  return 0;
}
