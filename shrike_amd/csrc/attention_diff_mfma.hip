// bfloat16 differential attention over the paged cache on the matrix units (gfx950): the kernels of
// attention_mfma.hip (single tokens with their keys split among wavefronts; prompt portions with a
// chunk of 32 keys shared in LDS) for heads of two maps over one set of values, for values of another
// size than keys, and for a window that keeps a sequence's first tokens.
//
// A key/value head's row in the key cache is D = maps * dim elements, [map 1, map 2].  A score of map
// m is the product of that row with a query whose elements outside map m are zero, so a map needs only
// the row's operand slices of 32 elements that its elements lie in (shared slices are masked in the
// query operand).  The products are formed transposed, S^T = K Q^T and O^T += V^T P^T: a lane owns
// a query, P is the second product's operand as it stands.
//
//   single tokens   a column of the products is (map, head): eight heads of two maps (or sixteen of
//                   one) meet a chunk's keys and values in one pass; keys and values are read once
//                   for both maps.
//   prompts         a wavefront owns 16 queries of one head, both maps: every value operand read
//                   from LDS serves both.
//
// The two maps meet where a head's sums are complete: at the end of the prompt kernel, or in
// diff_merge_kernel behind the single tokens' (and shared portions') partial results; there the
// difference is normed, scaled, multiplied by the head's gate, and rounded once.
#include "api.h"
#include "common.h"
#include "diff_mask.h"
#include "mfma_tile.h"

namespace shk {

namespace {

constexpr int kDiffSplits = 64;
constexpr int kDiffWaves = 4;  // wavefronts of the single-token kernel
// wavefronts of the prompt kernel: 16, or 8 where that many would make too few workgroups
constexpr int kDiffShared = 16, kDiffSharedSmall = 8;

struct DiffArgs {
  const bf16* q;  // [n][heads][D]
  bf16* out;      // [n][heads][DV]
  int heads, kv_heads;
  const int32_t* tables;
  int table_stride;
  const bf16* k_pool;  // [pages][kv_heads][D / 32][page_size][32]
  const bf16* v_pool;  // [pages][kv_heads][DV][page_size]
  PageDiv pd;
  int window, keep_first;
  float scale;
  float lambda, rest, eps;
  const float* gate;  // [n][heads] or null
  float* partial;
  int nsplit;
};

// The slices of a row that a map of DIM elements lies in: kSlices from first(m) on.
template <int DIM>
struct MapSlices {
  static constexpr int kSlices = (DIM + 31) / 32;
  static __device__ __forceinline__ constexpr int first(int m) { return m * DIM / 32; }
};

// ------------------------------------------------------------------ single tokens
// grid (kv_heads * blocks of heads, sequences, splits)
template <int D, int DV, int MAPS, bool NT>
__global__ void __launch_bounds__(kDiffWaves* kWave) diff_decode_kernel(const DiffArgs a, const int32_t* __restrict__ positions) {
  constexpr int DIM = D / MAPS, kCols = 16 / MAPS;
  constexpr int NBUF = 2;
  constexpr int kStep = kDiffWaves;  // chunks between two of one wavefront
  __shared__ float m_lds[kDiffWaves][16], l_lds[kDiffWaves][16];
  __shared__ float4 o_lds[kDiffWaves - 1][DV / 16][kWave];
  const int group = a.heads / a.kv_heads, blocks = (group + kCols - 1) / kCols;
  const int kvh = blockIdx.x / blocks, h0 = blockIdx.x % blocks * kCols;
  const int seq = blockIdx.y, z = blockIdx.z;
  const int wave = threadIdx.x / kWave;
  const int lane = threadIdx.x % kWave, j = lane % 16, g = lane / 16;
  const int map = j / kCols, hh = h0 + j % kCols;
  const bool live = hh < group;
  const int head = kvh * group + hh;
  const int ps = a.pd.ps;
  const int pos = positions[seq];
  const int lo = first_key(pos, a.window, 0);
  const KeptChunks kc(lo, a.keep_first);
  const int chunks = kc.count(pos);
  const int per = (chunks + a.nsplit - 1) / a.nsplit;
  const int c_begin = z * per + wave;
  const int c_end = (z + 1) * per < chunks ? (z + 1) * per : chunks;

  float m = -INFINITY, l = 0.f;  // base-2 logarithms; l is this lane's share of the sum until the end
  f32x4 o[DV / 16];              // element db*16 + 4*g + r of column j
#pragma unroll
  for (int db = 0; db < DV / 16; ++db) o[db] = f32x4{0.f, 0.f, 0.f, 0.f};

  if (c_begin < c_end) {
    struct Chunk {
      AFrag k[2][D / 32];
      AFrag v[DV / 16];
    };
    AFrag qf[D / 32];
    const bf16* qrow = a.q + (static_cast<size_t>(seq) * a.heads + (live ? head : kvh * group)) * D + g * 8;
#pragma unroll
    for (int ds = 0; ds < D / 32; ++ds) {
      qf[ds].u = make_uint4(0, 0, 0, 0);
      if (live && (ds * 32 + g * 8) / DIM == map) qf[ds].u = *reinterpret_cast<const uint4*>(qrow + ds * 32);
    }
    const float scale2 = a.scale * 1.4426950408889634f;
    const int32_t* table = a.tables + static_cast<size_t>(seq) * a.table_stride;
    const bool k_second = j >= 8, v_second = g >= 2;
    int k_lane[2];
#pragma unroll
    for (int t = 0; t < 2; ++t) k_lane[t] = (8 * ((j / 4) % 2) + 4 * t + j % 4) * 32 + g * 8;
    const int v_lane = j * ps + 8 * (g % 2);
    const size_t k_elems = static_cast<size_t>(ps) * D, v_elems = static_cast<size_t>(ps) * DV;

    auto fetch = [&](Chunk& c, int kb) {
      // pages of the chunk's two halves (the same for all lanes), clamped to ones that the sequence holds
      const int ka = held_key(kb, pos, lo, a.keep_first), kd = held_key(kb + 16, pos, lo, a.keep_first);
      const size_t page_a = static_cast<size_t>(table[__builtin_amdgcn_readfirstlane(a.pd.div(ka))]) * a.kv_heads + kvh;
      const size_t page_d = static_cast<size_t>(table[__builtin_amdgcn_readfirstlane(a.pd.div(kd))]) * a.kv_heads + kvh;
      const int slot_a = a.pd.mod(kb), slot_d = a.pd.mod(kb + 16);
      const bf16* krow = a.k_pool + (k_second ? page_d * k_elems + static_cast<size_t>(slot_d) * 32
                                              : page_a * k_elems + static_cast<size_t>(slot_a) * 32);
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int ds = 0; ds < D / 32; ++ds) {
          const bf16x8* at = reinterpret_cast<const bf16x8*>(krow + k_lane[t] + static_cast<size_t>(ds) * ps * 32);
          c.k[t][ds].v = NT ? __builtin_nontemporal_load(at) : *at;
        }
      const bf16* vcol = a.v_pool + (v_second ? page_d * v_elems + slot_d : page_a * v_elems + slot_a) + v_lane;
#pragma unroll
      for (int db = 0; db < DV / 16; ++db) {
        const bf16x8* at = reinterpret_cast<const bf16x8*>(vcol + static_cast<size_t>(db) * 16 * ps);
        c.v[db].v = NT ? __builtin_nontemporal_load(at) : *at;
      }
    };

    auto attend_chunk = [&](const Chunk& c, int kb, auto edge_tag) {
      constexpr bool edge = decltype(edge_tag)::value;
      f32x4 s[2];
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        s[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ds = 0; ds < D / 32; ++ds)
          s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(c.k[t][ds].v, qf[ds].v, s[t], 0, 0, 0);
      }
      float sc[8];  // keys kb + 8*g + e, e = 4*t + r
#pragma unroll
      for (int e = 0; e < 8; ++e) sc[e] = s[e / 4][e % 4] * scale2;
      const int g0 = kb + g * 8;
      uint4 keep_bits = make_uint4(~0u, ~0u, ~0u, ~0u);
      if (edge) {
        uint32_t w[4] = {0, 0, 0, 0};
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const bool in = reads_key(g0 + e, pos, lo, a.keep_first);
          if (!in) sc[e] = -INFINITY;
          // a masked key carries weight 0 but its slot may hold anything: it is zeroed, so that 0 * x stays 0
          if (in) w[e / 2] |= e % 2 ? 0xffff0000u : 0x0000ffffu;
        }
        keep_bits = make_uint4(w[0], w[1], w[2], w[3]);
      }
      float mx = max3(max3(sc[0], sc[1], sc[2]), max3(sc[3], sc[4], sc[5]), fmaxf(sc[6], sc[7]));
      mx = lanes4_max(mx);
      const float m_new = fmaxf(m, mx);
      const float m_safe = (m_new == -INFINITY) ? 0.f : m_new;
      const float alpha = __builtin_amdgcn_exp2f(m - m_safe);
      float pr[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) pr[e] = __builtin_amdgcn_exp2f(sc[e] - m_safe);
      l = l * alpha + (((pr[0] + pr[1]) + (pr[2] + pr[3])) + ((pr[4] + pr[5]) + (pr[6] + pr[7])));
      m = m_new;
      if (__builtin_amdgcn_ballot_w64(alpha != 1.f) != 0) {
#pragma unroll
        for (int db = 0; db < DV / 16; ++db) o[db] *= alpha;
      }
      AFrag pf;
#pragma unroll
      for (int e = 0; e < 8; ++e) pf.v[e] = static_cast<__bf16>(pr[e]);
#pragma unroll
      for (int db = 0; db < DV / 16; ++db) {
        AFrag vf = c.v[db];
        if (edge) {
          vf.u.x &= keep_bits.x;
          vf.u.y &= keep_bits.y;
          vf.u.z &= keep_bits.z;
          vf.u.w &= keep_bits.w;
        }
        o[db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf.v, pf.v, o[db], 0, 0, 0);
      }
    };
    auto attend = [&](const Chunk& c, int kb) {
      if (kb + 31 > pos || kb < lo)  // the same for all lanes
        attend_chunk(c, kb, EdgeTag<true>{});
      else
        attend_chunk(c, kb, EdgeTag<false>{});
    };

    // One chunk's loads are in flight while another is computed; past the end the last chunk's again (a step
    // without loads would make the compiler wait for all loads in flight at each step).
    const int c_last = c_begin + (c_end - 1 - c_begin) / kStep * kStep;
    Chunk buf[NBUF];
    fetch(buf[0], kc.key_of(c_begin));
    for (int c0 = c_begin; c0 < c_end; c0 += kStep * NBUF) {
#pragma unroll
      for (int u = 0; u < NBUF; ++u) {
        const int c = c0 + kStep * u;
        if (c >= c_end) break;
        fetch(buf[(u + 1) % NBUF], kc.key_of(c + kStep < c_last ? c + kStep : c_last));
        attend(buf[u], kc.key_of(c));
      }
    }
    l = lanes4_sum(l);
  }

  // the wavefronts' results become one: common maximum, sums in wavefront order
  if (g == 0) {
    m_lds[wave][j] = m;
    l_lds[wave][j] = l;
  }
  __syncthreads();
  float m_all = m_lds[0][j];
#pragma unroll
  for (int w = 1; w < kDiffWaves; ++w) m_all = fmaxf(m_all, m_lds[w][j]);
  const float m_ref = (m_all == -INFINITY) ? 0.f : m_all;
  l = 0.f;
#pragma unroll
  for (int w = 0; w < kDiffWaves; ++w) l += l_lds[w][j] * __builtin_amdgcn_exp2f(m_lds[w][j] - m_ref);
  const float mine = __builtin_amdgcn_exp2f(m - m_ref);
#pragma unroll
  for (int db = 0; db < DV / 16; ++db) o[db] *= mine;
  if (wave > 0) {
#pragma unroll
    for (int db = 0; db < DV / 16; ++db)
      o_lds[wave - 1][db][lane] = make_float4(o[db][0], o[db][1], o[db][2], o[db][3]);
  }
  __syncthreads();
  if (wave > 0 || !live) return;
#pragma unroll
  for (int w = 0; w < kDiffWaves - 1; ++w)
#pragma unroll
    for (int db = 0; db < DV / 16; ++db) {
      const float4 x = o_lds[w][db][lane];
      o[db][0] += x.x;
      o[db][1] += x.y;
      o[db][2] += x.z;
      o[db][3] += x.w;
    }
  // partial: O [token][head][map][split][DV], then (maximum, sum) [token][head][map][split][2]
  const size_t rows = static_cast<size_t>(gridDim.y) * a.heads * MAPS * a.nsplit;
  const size_t row = ((static_cast<size_t>(seq) * a.heads + head) * MAPS + map) * a.nsplit + z;
  float* dst = a.partial + row * DV + 4 * g;
#pragma unroll
  for (int db = 0; db < DV / 16; ++db)
    *reinterpret_cast<float4*>(dst + db * 16) = make_float4(o[db][0], o[db][1], o[db][2], o[db][3]);
  if (g == 0) *reinterpret_cast<float2*>(a.partial + rows * DV + row * 2) = make_float2(m_all, l);
}

// ------------------------------------------------------------------ partial results become heads
// One wavefront per (token, head): the splits of each map in order, the maps' difference, its norm, the gate.
// `first_token`: the token that the first partial row belongs to.
template <int DV, int MAPS>
__global__ void __launch_bounds__(kWave) diff_merge_kernel(const DiffArgs a, int first_token) {
  constexpr int NE = (DV + kWave - 1) / kWave;
  constexpr int kBatch = 8;  // splits in flight
  __shared__ float weight[MAPS][kDiffSplits];
  const int nsplit = a.nsplit;
  const size_t unit = blockIdx.x;  // token * heads + head
  const size_t rows = static_cast<size_t>(gridDim.x) * MAPS * nsplit;
  const int lane = threadIdx.x;
  float value[NE];
#pragma unroll
  for (int map = 0; map < MAPS; ++map) {
    const size_t row = (unit * MAPS + map) * nsplit;
    const float* src = a.partial + row * DV;
    float2 mine = make_float2(-INFINITY, 0.f);
    if (lane < nsplit) mine = *reinterpret_cast<const float2*>(a.partial + rows * DV + (row + lane) * 2);
    float x[kBatch][NE];
    auto fetch = [&](int z0) {
#pragma unroll
      for (int u = 0; u < kBatch; ++u)
#pragma unroll
        for (int e = 0; e < NE; ++e) {
          const int d = lane + e * kWave;
          x[u][e] = (z0 + u < nsplit && d < DV) ? src[static_cast<size_t>(z0 + u) * DV + d] : 0.f;
        }
    };
    fetch(0);  // travels while the weights are formed
    const float mx = wave_max(mine.x);
    const float w = mine.x == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(mine.x - mx);
    weight[map][lane] = w;
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    const float wl = w * mine.y;
    float den = 0.f;
    for (int zz = 0; zz < nsplit; ++zz) den += __shfl(wl, zz, kWave);
    float acc[NE];
#pragma unroll
    for (int e = 0; e < NE; ++e) acc[e] = 0.f;
    for (int z0 = 0; z0 < nsplit; z0 += kBatch) {
#pragma unroll
      for (int u = 0; u < kBatch; ++u) {
        const float wz = z0 + u < nsplit ? weight[map][z0 + u] : 0.f;
#pragma unroll
        for (int e = 0; e < NE; ++e) acc[e] += wz * x[u][e];
      }
      if (z0 + kBatch < nsplit) fetch(z0 + kBatch);
    }
    const float inv = 1.f / den;
#pragma unroll
    for (int e = 0; e < NE; ++e) value[e] = map == 0 ? acc[e] * inv : value[e] - a.lambda * (acc[e] * inv);
  }
  float mult = a.gate ? a.gate[static_cast<size_t>(first_token) * a.heads + unit] : 1.f;
  if (MAPS == 2) {
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < NE; ++e)
      if (lane + e * kWave < DV) ss = fmaf(value[e], value[e], ss);
    mult *= a.rest / sqrtf(wave_sum(ss) / static_cast<float>(DV) + a.eps);
  }
#pragma unroll
  for (int e = 0; e < NE; ++e) {
    const int d = lane + e * kWave;
    if (d < DV) a.out[(static_cast<size_t>(first_token) * a.heads + unit) * DV + d] = from_float<bf16>(value[e] * mult);
  }
}

// ------------------------------------------------------------------ prompt portions
// A workgroup of WAVES wavefronts serves every query head of one key/value head for a run of 16 * tiles
// queries of one sequence; wavefront w owns head w % group, query tile w / group, both maps.  The chunk
// of 32 keys (all of the row's slices, and the values) is staged once in LDS in operand layout.
// Two maps' sums take twice the registers of one: with 8 wavefronts a workgroup they get 256 each (two
// wavefronts on a SIMD, whose two maps are two independent chains); held to 128 the kernel spills and
// takes 2.7 times as long (28 heads over 4, maps of 64, 2,048 queries: 305 us against 113), which is
// what more than 8 heads a key/value head, in 16 wavefronts, still have to live with.
// grid: entries of wg_seq / wg_q0 x kv_heads x splits.
template <int D, int DV, int MAPS, int WAVES>
__global__ void __launch_bounds__(WAVES* kWave) __attribute__((amdgpu_waves_per_eu(WAVES >= 16 || MAPS == 1 ? 4 : 2)))
    diff_prefill_kernel(const DiffArgs a, int tiles, const int32_t* __restrict__ cu_q,
                        const int32_t* __restrict__ ctx_lens, const int32_t* __restrict__ wg_seq,
                        const int32_t* __restrict__ wg_q0, int first_token, int partial_rows) {
  constexpr int DIM = D / MAPS;
  constexpr int NS = MapSlices<DIM>::kSlices;
  constexpr int kKFrags = 2 * (D / 32), kVFrags = DV / 16, kFrags = kKFrags + kVFrags;
  constexpr int kPer = (kFrags + WAVES - 1) / WAVES;  // fragments each wavefront stages
  typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));
  __shared__ u32x4 kv[2][kFrags][kWave];

  const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
  const int j = lane % 16, g = lane / 16;
  const int ps = a.pd.ps, nsplit = a.nsplit;
  const int z = blockIdx.x % nsplit;  // which share of the entry's keys
  const int wg = blockIdx.x / (nsplit * a.kv_heads), kvh = (blockIdx.x / nsplit) % a.kv_heads;
  const int seq = wg_seq[wg], q0 = wg_q0[wg];
  const int group = a.heads / a.kv_heads;
  const int tok0 = cu_q[seq], q_len = cu_q[seq + 1] - tok0;
  const int start = ctx_lens[seq] - q_len;
  const int q_end = (q0 + 16 * tiles < q_len) ? q0 + 16 * tiles : q_len;
  const size_t k_elems = static_cast<size_t>(ps) * D, v_elems = static_cast<size_t>(ps) * DV;
  const int32_t* table = a.tables + static_cast<size_t>(seq) * a.table_stride;

  // bounds over the whole workgroup: what has to be staged
  const int pos_min = start + q0, pos_max = start + q_end - 1;
  const int lo_min = first_key(pos_min, a.window, 0), lo_max = first_key(pos_max, a.window, 0);
  const KeptChunks kc(lo_min, a.keep_first);
  const int nchunks = kc.count(pos_max);
  const int per_split = (nchunks + nsplit - 1) / nsplit;
  const int c_first = z * per_split;
  const int c_end = c_first + per_split < nchunks ? c_first + per_split : nchunks;

  // this wavefront's head and queries; a lane owns query j
  const int unit_q0 = q0 + (wave / group) * 16;
  const bool valid = wave < tiles * group && unit_q0 < q_len;
  const int head = kvh * group + wave % group;
  const int rows = !valid ? 0 : (q_len - unit_q0 < 16 ? q_len - unit_q0 : 16);
  AFrag qf[MAPS][NS];
  {
    const bf16* qrow = a.q + (static_cast<size_t>(tok0 + (valid ? unit_q0 + (j < rows ? j : 0) : 0)) * a.heads + head) * D + g * 8;
#pragma unroll
    for (int mp = 0; mp < MAPS; ++mp)
#pragma unroll
      for (int ds = 0; ds < NS; ++ds) {
        const int slice = MapSlices<DIM>::first(mp) + ds;
        qf[mp][ds].u = make_uint4(0, 0, 0, 0);
        if (j < rows && (slice * 32 + g * 8) / DIM == mp) qf[mp][ds].u = *reinterpret_cast<const uint4*>(qrow + slice * 32);
      }
  }
  const int q_pos = j < rows ? start + unit_q0 + j : -1;
  const int q_lo = first_key(q_pos, a.window, 0);
  float m[MAPS], l[MAPS];
  f32x4 o[MAPS][DV / 16];
#pragma unroll
  for (int mp = 0; mp < MAPS; ++mp) {
    m[mp] = -INFINITY, l[mp] = 0.f;
#pragma unroll
    for (int db = 0; db < DV / 16; ++db) o[mp][db] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const float scale2 = a.scale * 1.4426950408889634f;

  // staging: wavefront w fetches fragments w, w + WAVES, ...; fragment f < kKFrags is K tile f / (D/32),
  // slice f % (D/32), row i of K tile t being key 8*(i/4) + 4*t + i%4 of the chunk; the others are V^T
  // blocks of 16 elements.  Every load is unconditional.
  const bool second_k = j >= 8, second_v = g >= 2;
  int lane_off[kPer];
  bool is_k[kPer];
#pragma unroll
  for (int i = 0; i < kPer; ++i) {
    const int f = (wave + WAVES * i) % kFrags;
    is_k[i] = f < kKFrags;
    if (is_k[i]) {
      const int t = f / (D / 32), ds = f % (D / 32);
      lane_off[i] = (8 * ((j / 4) % 2) + 4 * t + j % 4) * 32 + ds * ps * 32 + g * 8;
    } else {
      lane_off[i] = ((f - kKFrags) * 16 + j) * ps + 8 * (g % 2);
    }
  }
  auto fetch = [&](u32x4 (&held)[kPer], int chunk) {
    const int kb = kc.key_of(chunk < nchunks ? chunk : nchunks - 1);
    const int ka = held_key(kb, pos_max, lo_min, a.keep_first), kd = held_key(kb + 16, pos_max, lo_min, a.keep_first);
    const size_t page_a = static_cast<size_t>(table[__builtin_amdgcn_readfirstlane(a.pd.div(ka))]) * a.kv_heads + kvh;
    const size_t page_d = static_cast<size_t>(table[__builtin_amdgcn_readfirstlane(a.pd.div(kd))]) * a.kv_heads + kvh;
    const int slot_a = a.pd.mod(kb), slot_d = a.pd.mod(kb + 16);
    const bf16* krow = a.k_pool + (second_k ? page_d * k_elems + static_cast<size_t>(slot_d) * 32
                                            : page_a * k_elems + static_cast<size_t>(slot_a) * 32);
    const bf16* vcol = a.v_pool + (second_v ? page_d * v_elems + slot_d : page_a * v_elems + slot_a);
#pragma unroll
    for (int i = 0; i < kPer; ++i) held[i] = *reinterpret_cast<const u32x4*>((is_k[i] ? krow : vcol) + lane_off[i]);
    __builtin_amdgcn_sched_barrier(0);  // the loads go out before the multiplications
  };
  auto put = [&](const u32x4 (&held)[kPer], int chunk, int buf) {
    const int kb = kc.key_of(chunk);
    const int g0 = kb + g * 8;  // a V fragment's lane holds keys g0 .. g0 + 7
#pragma unroll
    for (int i = 0; i < kPer; ++i) {
      u32x4 x = held[i];
      // keys that no query of the workgroup reads carry weight 0, but their slots may hold anything
      if (!is_k[i] && (kb < lo_min || kb + 31 > pos_max)) {
        asm volatile("");  // stays a branch: as selects the comparisons would run for every chunk
        u32x4 keep;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const bool p = reads_key(g0 + 2 * e, pos_max, lo_min, a.keep_first);
          const bool r = reads_key(g0 + 2 * e + 1, pos_max, lo_min, a.keep_first);
          keep[e] = (p ? 0x0000ffffu : 0u) | (r ? 0xffff0000u : 0u);
        }
        x &= keep;
      }
      kv[buf][(wave + WAVES * i) % kFrags][lane] = x;
    }
  };
  auto attend = [&](int buf, int chunk) {
    const int kb = kc.key_of(chunk);
    const int g0 = kb + g * 8;
    // (wave-uniform) some query of the workgroup does not read the whole chunk
    const bool edge = kb + 31 > pos_min || (kb < lo_max && kb + 31 >= a.keep_first);
    AFrag pf[MAPS];
#pragma unroll
    for (int mp = 0; mp < MAPS; ++mp) {
      f32x4 s[2];
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        s[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ds = 0; ds < NS; ++ds)
          s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              __builtin_bit_cast(bf16x8, kv[buf][t * (D / 32) + MapSlices<DIM>::first(mp) + ds][lane]), qf[mp][ds].v, s[t], 0, 0, 0);
      }
      float sc[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) sc[e] = s[e / 4][e % 4] * scale2;
      if (edge) {
        asm volatile("");  // stays a branch
#pragma unroll
        for (int e = 0; e < 8; ++e)
          if (!reads_key(g0 + e, q_pos, q_lo, a.keep_first)) sc[e] = -INFINITY;
      }
      float mx = max3(max3(sc[0], sc[1], sc[2]), max3(sc[3], sc[4], sc[5]), fmaxf(sc[6], sc[7]));
      mx = lanes4_max(mx);
      const float m_new = fmaxf(m[mp], mx);
      const float m_safe = (m_new == -INFINITY) ? 0.f : m_new;
      const float alpha = __builtin_amdgcn_exp2f(m[mp] - m_safe);
      float pr[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) pr[e] = __builtin_amdgcn_exp2f(sc[e] - m_safe);
      l[mp] = l[mp] * alpha + (((pr[0] + pr[1]) + (pr[2] + pr[3])) + ((pr[4] + pr[5]) + (pr[6] + pr[7])));
      m[mp] = m_new;
      if (__builtin_amdgcn_ballot_w64(alpha != 1.f) != 0) {  // some query's maximum rose
#pragma unroll
        for (int db = 0; db < DV / 16; ++db) o[mp][db] *= alpha;
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) pf[mp].v[e] = static_cast<__bf16>(pr[e]);
    }
#pragma unroll
    for (int db = 0; db < DV / 16; ++db) {
      const bf16x8 vf = __builtin_bit_cast(bf16x8, kv[buf][kKFrags + db][lane]);
#pragma unroll
      for (int mp = 0; mp < MAPS; ++mp) o[mp][db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[mp].v, o[mp][db], 0, 0, 0);
    }
  };

  // chunk c is multiplied from LDS buffer (c - c_first) % 2 while the loads of the next two are in flight
  if (c_first < c_end) {  // the same for every wavefront of the workgroup
    u32x4 even[kPer], odd[kPer];
    fetch(even, c_first);
    fetch(odd, c_first + 1);
    put(even, c_first, 0);
    __syncthreads();
    int c = c_first;
    for (; c + 2 < c_end; c += 2) {
      fetch(even, c + 2);
      attend(0, c);
      put(odd, c + 1, 1);
      __syncthreads();
      fetch(odd, c + 3);
      attend(1, c + 1);
      put(even, c + 2, 0);
      __syncthreads();
    }
    attend(0, c);
    if (c + 1 < c_end) {
      put(odd, c + 1, 1);
      __syncthreads();
      attend(1, c + 1);
    }
  }

#pragma unroll
  for (int mp = 0; mp < MAPS; ++mp) l[mp] = lanes4_sum(l[mp]);
  const size_t token = static_cast<size_t>(tok0) + unit_q0 + j;
  if (nsplit > 1) {
    if (j >= rows) return;
    // a share's results, for diff_merge_kernel; rows count from the step's first prompt token
#pragma unroll
    for (int mp = 0; mp < MAPS; ++mp) {
      const size_t row = (((token - first_token) * a.heads + head) * MAPS + mp) * nsplit + z;
      float* dst = a.partial + row * DV + 4 * g;
#pragma unroll
      for (int db = 0; db < DV / 16; ++db)
        *reinterpret_cast<float4*>(dst + db * 16) = make_float4(o[mp][db][0], o[mp][db][1], o[mp][db][2], o[mp][db][3]);
      if (g == 0)
        *reinterpret_cast<float2*>(a.partial + static_cast<size_t>(partial_rows) * MAPS * nsplit * DV + row * 2) =
            make_float2(m[mp], l[mp]);
    }
    return;
  }
  float inv[MAPS];
#pragma unroll
  for (int mp = 0; mp < MAPS; ++mp) inv[mp] = 1.f / l[mp];
  float ss = 0.f;
#pragma unroll
  for (int db = 0; db < DV / 16; ++db)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      float v = o[0][db][r] * inv[0];
      if (MAPS == 2) v -= a.lambda * (o[MAPS - 1][db][r] * inv[MAPS - 1]);
      o[0][db][r] = v;
      ss = fmaf(v, v, ss);
    }
  float mult = 1.f;
  if (MAPS == 2) mult = a.rest / sqrtf(lanes4_sum(ss) / static_cast<float>(DV) + a.eps);
  if (j >= rows) return;
  if (a.gate) mult *= a.gate[token * a.heads + head];
  bf16* dst = a.out + (token * a.heads + head) * DV + 4 * g;
#pragma unroll
  for (int db = 0; db < DV / 16; ++db) {
    uint2 packed;
    packed.x = bf16_bits(o[0][db][0] * mult) | (static_cast<uint32_t>(bf16_bits(o[0][db][1] * mult)) << 16);
    packed.y = bf16_bits(o[0][db][2] * mult) | (static_cast<uint32_t>(bf16_bits(o[0][db][3] * mult)) << 16);
    *reinterpret_cast<uint2*>(dst + db * 16) = packed;
  }
}

// ------------------------------------------------------------------ dispatch by sizes

bool takes(int maps, int row_dim, int v_dim) {
  const bool sizes = row_dim % 32 == 0 && row_dim >= 32 && row_dim <= 128 && v_dim % 32 == 0 && v_dim >= 32 && v_dim <= 128;
  return sizes && (maps == 2 || (maps == 1 && row_dim == v_dim));
}

// CALL(D, DV, MAPS) for the kernels' sizes
#define SHK_DIFF_V(CALL, D)                     \
  switch (v_dim) {                              \
    case 32: CALL(D, 32, 2); break;             \
    case 64: CALL(D, 64, 2); break;             \
    case 96: CALL(D, 96, 2); break;             \
    default: CALL(D, 128, 2); break;            \
  }
#define SHK_DIFF_SIZES(CALL)                    \
  if (maps == 2) {                              \
    switch (row_dim) {                          \
      case 32: SHK_DIFF_V(CALL, 32) break;      \
      case 64: SHK_DIFF_V(CALL, 64) break;      \
      case 96: SHK_DIFF_V(CALL, 96) break;      \
      default: SHK_DIFF_V(CALL, 128) break;     \
    }                                           \
  } else {                                      \
    switch (row_dim) {                          \
      case 32: CALL(32, 32, 1); break;          \
      case 64: CALL(64, 64, 1); break;          \
      case 96: CALL(96, 96, 1); break;          \
      default: CALL(128, 128, 1); break;        \
    }                                           \
  }

template <int DV, int MAPS>
void launch_merge(const DiffArgs& a, int tokens, int first_token, hipStream_t s) {
  diff_merge_kernel<DV, MAPS><<<tokens * a.heads, kWave, 0, s>>>(a, first_token);
}

int check_diff(const char* who, const DiffArgs& a, int maps, int row_dim, int v_dim) {
  SHK_REQUIRE(a.heads > 0 && a.kv_heads > 0 && a.heads % a.kv_heads == 0,
              "%s: heads=%d must be a positive multiple of kv_heads=%d", who, a.heads, a.kv_heads);
  SHK_REQUIRE(takes(maps, row_dim, v_dim), "%s: %d maps with rows of %d and values of %d are not served", who, maps, row_dim,
              v_dim);
  SHK_REQUIRE(a.pd.ps > 0 && a.pd.ps % 16 == 0, "%s: page_size %d is not a multiple of 16", who, a.pd.ps);
  SHK_REQUIRE(a.window >= 0 && a.keep_first >= 0, "%s: bad mask window=%d keep_first=%d", who, a.window, a.keep_first);
  SHK_REQUIRE(a.nsplit >= 1 && a.nsplit <= kDiffSplits, "%s: %d key splits (at most %d)", who, a.nsplit, kDiffSplits);
  SHK_REQUIRE(a.q && a.out && a.tables && a.k_pool && a.v_pool && a.table_stride > 0, "%s: null pointer", who);
  SHK_REQUIRE(reinterpret_cast<uintptr_t>(a.q) % 16 == 0 && reinterpret_cast<uintptr_t>(a.out) % 8 == 0 &&
                  reinterpret_cast<uintptr_t>(a.partial) % 16 == 0,
              "%s: q and partial must be 16-byte and out 8-byte aligned", who);
  SHK_REQUIRE(static_cast<long long>(a.table_stride) * a.pd.ps * a.pd.ps < (1ll << 32),
              "%s: a block table of %d pages of %d is beyond the kernel's range", who, a.table_stride, a.pd.ps);
  return 0;
}

DiffArgs diff_args(const void* q, void* out, int heads, int kv_heads, const int32_t* tables, int table_stride,
                   const void* k_pool, const void* v_pool, int page_size, int window, int keep_first, float scale,
                   float lambda, float rest, float eps, const float* gate, float* partial, int nsplit) {
  DiffArgs a;
  a.q = static_cast<const bf16*>(q), a.out = static_cast<bf16*>(out), a.heads = heads, a.kv_heads = kv_heads;
  a.tables = tables, a.table_stride = table_stride;
  a.k_pool = static_cast<const bf16*>(k_pool), a.v_pool = static_cast<const bf16*>(v_pool);
  a.pd = PageDiv{page_size, page_size > 0 ? static_cast<uint32_t>(((1ull << 32) + page_size - 1) / page_size) : 0u};
  a.window = window, a.keep_first = keep_first, a.scale = scale, a.lambda = lambda, a.rest = rest, a.eps = eps;
  a.gate = gate, a.partial = partial, a.nsplit = nsplit;
  return a;
}

}  // namespace

}  // namespace shk

using namespace shk;

extern "C" int shk_diff_attention_supports_mfma(int heads, int kv_heads, int maps, int row_dim, int v_dim, int page_size) {
  return heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && heads / kv_heads <= kDiffShared && takes(maps, row_dim, v_dim) &&
         page_size > 0 && page_size % 16 == 0;
}

// Query tiles of 16 that one workgroup of the prompt kernel serves (0: the shape is not served).
extern "C" int shk_diff_attention_tiles(int heads, int kv_heads, int small) {
  const int group = kv_heads > 0 ? heads / kv_heads : 0, units = small ? kDiffSharedSmall : kDiffShared;
  return group < 1 || group > units ? 0 : units / group;
}

extern "C" int shk_diff_attention_decode_bf16(const void* q, void* out, int num_seqs, int heads, int kv_heads, int maps,
                                              int row_dim, int v_dim, const int32_t* positions, const int32_t* tables,
                                              int table_stride, const void* k_pool, const void* v_pool, int page_size,
                                              int window, int keep_first, float scale, float lambda, float rest, float eps,
                                              const float* gate, float* partial, int nsplit, int streaming, void* stream) {
  const DiffArgs a = diff_args(q, out, heads, kv_heads, tables, table_stride, k_pool, v_pool, page_size, window, keep_first,
                               scale, lambda, rest, eps, gate, partial, nsplit);
  if (num_seqs == 0) return 0;
  if (check_diff("diff_attention_decode", a, maps, row_dim, v_dim)) return 1;
  SHK_REQUIRE(num_seqs > 0 && num_seqs <= 65535 && positions && partial, "diff_attention_decode: bad arguments");
  hipStream_t s = static_cast<hipStream_t>(stream);
  const int cols = 16 / maps, group = heads / kv_heads;
  const dim3 grid(kv_heads * ((group + cols - 1) / cols), num_seqs, nsplit);
#define SHK_CALL(D, DV, MAPS)                                                                      \
  do {                                                                                             \
    if (streaming) diff_decode_kernel<D, DV, MAPS, true><<<grid, kDiffWaves * kWave, 0, s>>>(a, positions);  \
    else diff_decode_kernel<D, DV, MAPS, false><<<grid, kDiffWaves * kWave, 0, s>>>(a, positions);           \
    launch_merge<DV, MAPS>(a, num_seqs, 0, s);                                                     \
  } while (0)
  SHK_DIFF_SIZES(SHK_CALL)
#undef SHK_CALL
  SHK_LAUNCH_CHECK("diff_attention_decode");
  return 0;
}

extern "C" int shk_diff_attention_prefill_bf16(const void* q, void* out, int num_wgs, int heads, int kv_heads, int maps,
                                               int row_dim, int v_dim, const int32_t* cu_q, const int32_t* ctx_lens,
                                               const int32_t* wg_lists, const int32_t* tables, int table_stride,
                                               const void* k_pool, const void* v_pool, int page_size, int window,
                                               int keep_first, float scale, float lambda, float rest, float eps,
                                               const float* gate, int small, float* partial, int nsplit, int first_token,
                                               int prompt_tokens, void* stream) {
  const DiffArgs a = diff_args(q, out, heads, kv_heads, tables, table_stride, k_pool, v_pool, page_size, window, keep_first,
                               scale, lambda, rest, eps, gate, partial, nsplit);
  if (num_wgs == 0) return 0;
  if (check_diff("diff_attention_prefill", a, maps, row_dim, v_dim)) return 1;
  const int tiles = shk_diff_attention_tiles(heads, kv_heads, small);
  SHK_REQUIRE(tiles > 0, "diff_attention_prefill: %d query heads per key/value head are not served", heads / kv_heads);
  SHK_REQUIRE(num_wgs > 0 && static_cast<long long>(num_wgs) * kv_heads * nsplit < (1ll << 31) && cu_q && ctx_lens && wg_lists,
              "diff_attention_prefill: bad arguments");
  SHK_REQUIRE(nsplit == 1 || (partial && first_token >= 0 && prompt_tokens > 0 &&
                              static_cast<long long>(prompt_tokens) * heads < (1ll << 31)),
              "diff_attention_prefill: key splits need a partial buffer, the index of the first prompt token and the number of "
              "prompt tokens");
  hipStream_t s = static_cast<hipStream_t>(stream);
  const dim3 grid(num_wgs * kv_heads * nsplit);
  const int rows = prompt_tokens * heads;
#define SHK_CALL(D, DV, MAPS)                                                                                    \
  do {                                                                                                           \
    if (small)                                                                                                   \
      diff_prefill_kernel<D, DV, MAPS, kDiffSharedSmall><<<grid, kDiffSharedSmall * kWave, 0, s>>>(              \
          a, tiles, cu_q, ctx_lens, wg_lists, wg_lists + num_wgs, first_token, rows);                            \
    else                                                                                                         \
      diff_prefill_kernel<D, DV, MAPS, kDiffShared><<<grid, kDiffShared * kWave, 0, s>>>(                        \
          a, tiles, cu_q, ctx_lens, wg_lists, wg_lists + num_wgs, first_token, rows);                            \
    if (nsplit > 1) launch_merge<DV, MAPS>(a, prompt_tokens, first_token, s);                                    \
  } while (0)
  SHK_DIFF_SIZES(SHK_CALL)
#undef SHK_CALL
  SHK_LAUNCH_CHECK("diff_attention_prefill");
  return 0;
}
