// What stands between the projections of an attention layer with a short convolution and its
// attention kernels, in one pass: a causal convolution over time on every channel of queries, keys and
// values, the rotation of queries and keys, keys and values into their cache pages, the queries into a
// tensor of their own, the heads' gates through a sigmoid, and the convolution's last inputs into the
// request's state slot.
//
// A row of the projections is [queries: q_heads * dim | keys: k_heads * dim | values: v_heads * v_dim |
// gates | padding] (a layer that reads another layer's cache: [queries | gates | padding]), in the
// compute dtype, or as the float32 partial sums of a product split along k (added here, in order,
// with the bias).  `maps` neighbouring key heads share one row of the key cache: key head u is part u %
// maps of the row of cache head u / maps.
//
// A workgroup takes a tile of consecutive tokens of one sequence: single tokens a tile each, prompt
// portions in tiles of kTile.  A thread owns a run of V channels (for rotated elements the run and its
// partner half a rotation away) and walks the tile's tokens with the convolution's window in registers.
// Inputs before the tile come from the step's own rows where the portion reaches that far back, else from
// the state slot, which holds the last taps - 1 inputs of the sequence, oldest first [taps - 1][channels]
// in float32; before the sequence's start they are zero.  The tile with the portion's first token is the
// only one that reads the slot (tiles hold at least taps - 1 tokens), and the same threads write it back,
// so no two workgroups meet there.
#include "api.h"
#include "common.h"

namespace shk {

namespace {

constexpr int kConvThreads = 256;
constexpr int kTile = 8;        // tokens of a prompt portion a workgroup walks
constexpr int kMaxTaps = 33;
constexpr int kMaxRotHalf = 128;

struct ConvStore {
  const void* proj;
  int ldp;
  const float* parts;
  int splits;
  size_t part_stride;
  const float* bias;
  const float* taps;  // [taps][channels], or null: no convolution
  int K;
  int q_heads, k_heads, dim, rot_dim, v_heads, v_dim, gates, maps;
  const float* inv_freq;
  float magnitude;
  const int32_t* positions;
  const int32_t* cu_q;
  const int32_t* slots;
  const int32_t* tables;
  int table_stride;
  float* state;
  long long slot_stride;
  int num_single;
  const int32_t* tile_seq;
  const int32_t* tile_q0;
  int tile;
  void* q_out;
  float* gate_out;
  void* k_pool;
  void* v_pool;
  int page_size, num_pages;
};

template <typename T, int V>
__device__ __forceinline__ void put_run(T* p, const float (&x)[V]) {
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

// V neighbouring floats
template <int V>
__device__ __forceinline__ void get_floats(const float* p, float (&x)[V]) {
  if constexpr (V == 1) {
    x[0] = p[0];
  } else {
    const float4 a = *reinterpret_cast<const float4*>(p);
    x[0] = a.x, x[1] = a.y, x[2] = a.z, x[3] = a.w;
  }
}

// the projections' columns col .. col + V - 1 of row t
template <typename T, int V>
__device__ __forceinline__ void fetch(const ConvStore& a, size_t t, int col, float (&x)[V]) {
  if (a.splits == 0) {
    const T* p = static_cast<const T*>(a.proj) + t * a.ldp + col;
    if constexpr (V == 1) {
      x[0] = to_float(p[0]);
    } else if constexpr (sizeof(T) == 4) {
      get_floats<V>(reinterpret_cast<const float*>(p), x);
    } else {
      const uint2 u = *reinterpret_cast<const uint2*>(p);
      x[0] = __uint_as_float(u.x << 16), x[1] = __uint_as_float(u.x & 0xffff0000u);
      x[2] = __uint_as_float(u.y << 16), x[3] = __uint_as_float(u.y & 0xffff0000u);
    }
    return;
  }
  const float* p = a.parts + t * a.ldp + col;
#pragma unroll
  for (int e = 0; e < V; ++e) x[e] = 0.f;
  for (int z0 = 0; z0 < a.splits; z0 += 4) {  // four parts in flight, added in order
    float more[4][V];
#pragma unroll
    for (int u = 0; u < 4; ++u)
      get_floats<V>(p + static_cast<size_t>(z0 + u < a.splits ? z0 + u : a.splits - 1) * a.part_stride, more[u]);
#pragma unroll
    for (int u = 0; u < 4; ++u)
      if (z0 + u < a.splits) {
#pragma unroll
        for (int e = 0; e < V; ++e) x[e] += more[u][e];
      }
  }
  if (a.bias) {
#pragma unroll
    for (int e = 0; e < V; ++e) x[e] += a.bias[col + e];
  }
}

// KT: the number of taps where the window is held in registers (1 where there is no convolution), 0:
// any number, inputs read again for every token.  TOK: tokens a tile at most (KT > 0).
template <typename T, int V, int KT, int TOK>
__global__ void __launch_bounds__(kConvThreads) conv_store_kernel(const ConvStore a) {
  extern __shared__ float turns[];  // [tile][half][2]: cosine and sine times the magnitude
  const bool single = static_cast<int>(blockIdx.x) < a.num_single;
  const int seq = single ? blockIdx.x : a.tile_seq[blockIdx.x - a.num_single];
  const int q0 = single ? 0 : a.tile_q0[blockIdx.x - a.num_single];
  const int first = a.cu_q[seq], len = a.cu_q[seq + 1] - first;
  const int count = len - q0 < a.tile ? len - q0 : a.tile;
  const int start = a.positions[first];  // position of the portion's first token
  const int half = a.rot_dim / 2, tail = a.dim - a.rot_dim;
  const int K = KT > 0 ? KT : a.K;

  // what this thread owns
  const int turned = (a.q_heads + a.k_heads) * (half / V), plain = (a.q_heads + a.k_heads) * (tail / V);
  const int values = a.v_heads * a.v_dim / V;
  const int item = blockIdx.y * kConvThreads + threadIdx.x;
  enum { kTurned, kPlain, kValue, kGate, kNone } role = kNone;
  int u = 0, i = 0, col = 0;  // head, element within it, column
  if (item < turned) {
    role = kTurned;
    u = item / (half / V), i = item % (half / V) * V;
    col = u * a.dim + i;
  } else if (item < turned + plain) {
    role = kPlain;
    u = (item - turned) / (tail / V), i = a.rot_dim + (item - turned) % (tail / V) * V;
    col = u * a.dim + i;
  } else if (item < turned + plain + values) {
    role = kValue;
    i = (item - turned - plain) * V;
    col = (a.q_heads + a.k_heads) * a.dim + i;
  } else if (item < turned + plain + values + a.gates) {
    role = kGate;
    i = item - turned - plain - values;
    col = (a.q_heads + a.k_heads) * a.dim + a.v_heads * a.v_dim + i;
  }
  const int channels = (a.q_heads + a.k_heads) * a.dim + a.v_heads * a.v_dim;
  float* slot = a.taps && K > 1 ? a.state + static_cast<size_t>(a.slots[seq]) * a.slot_stride : nullptr;

  for (int f = threadIdx.x; f < count * half; f += kConvThreads) {
    // the angle is a float32 product; it reaches thousands of radians and is brought into [-pi, pi] in
    // float64 (exact to 1e-13) before the float32 sine and cosine
    const float angle = static_cast<float>(start + q0 + f / half) * a.inv_freq[f % half];
    const double wide = static_cast<double>(angle);
    const double whole = rint(wide * 0.15915494309189535);
    float sv, cv;
    sincosf(static_cast<float>(fma(whole, -6.283185307179586, wide)), &sv, &cv);
    turns[2 * f] = cv * a.magnitude;
    turns[2 * f + 1] = sv * a.magnitude;
  }
  __syncthreads();
  if (role == kNone) return;
  if (role == kGate) {
    for (int k = 0; k < count; ++k) {
      const size_t t = static_cast<size_t>(first) + q0 + k;
      float x[1];
      fetch<T, 1>(a, t, col, x);
      a.gate_out[t * a.gates + i] = 1.f / (1.f + expf(-x[0]));
    }
    return;
  }

  // the input of channels c .. c + V - 1 at row r of the portion (r < 0: before it)
  auto input = [&](int r, int c, float (&x)[V]) {
    if (r >= 0) {
      fetch<T, V>(a, static_cast<size_t>(first) + r, c, x);
    } else if (slot && start + r >= 0) {
      get_floats<V>(slot + static_cast<size_t>(K - 1 + r) * channels + c, x);
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e) x[e] = 0.f;
    }
  };
  const int step = half;  // from a turned run to its partner

  // the convolved run(s) of the tile's token k, turned and written
  auto finish = [&](int k, float (&y)[V], float (&z)[V]) {
    const int pos = start + q0 + k;
    const size_t t = static_cast<size_t>(first) + q0 + k;
    if (role == kTurned) {
      const float* cs = turns + 2 * (static_cast<size_t>(k) * half + i);
#pragma unroll
      for (int e = 0; e < V; ++e) {
        const float c = cs[2 * e], s = cs[2 * e + 1];
        const float p = y[e] * c - z[e] * s, q = z[e] * c + y[e] * s;
        y[e] = p, z[e] = q;
      }
    }
    if (role != kValue && u < a.q_heads) {
      T* dst = static_cast<T*>(a.q_out) + t * (static_cast<size_t>(a.q_heads) * a.dim) + u * a.dim + i;
      put_run<T, V>(dst, y);
      if (role == kTurned) put_run<T, V>(dst + step, z);
      return;
    }
    const int page = a.tables[static_cast<size_t>(seq) * a.table_stride + pos / a.page_size];
    if (page < 0 || page >= a.num_pages) return;  // a host bug; never dereferenced
    const int place = pos % a.page_size;
    if (role == kValue) {
      T* dst = static_cast<T*>(a.v_pool) + (static_cast<size_t>(page) * a.v_heads * a.v_dim + i) * a.page_size + place;
#pragma unroll
      for (int e = 0; e < V; ++e) dst[static_cast<size_t>(e) * a.page_size] = from_float<T>(y[e]);
      return;
    }
    const int kh = u - a.q_heads, g = kh / a.maps, width = a.maps * a.dim;
    const int d = kh % a.maps * a.dim + i;  // element of the cached row
    T* dst = static_cast<T*>(a.k_pool) +
             (static_cast<size_t>(page) * (a.k_heads / a.maps) + g) * a.page_size * width;
    // (runs of four lie within one slab: slabs are 32 elements or the whole row)
    put_run<T, V>(dst + key_offset(place, d, a.page_size, width), y);
    if (role == kTurned) put_run<T, V>(dst + key_offset(place, d + step, a.page_size, width), z);
  };

  if constexpr (KT > 0) {
    constexpr int kRows = TOK + KT - 1;
    float x[kRows][V], x2[kRows][V];
    const bool two = role == kTurned;
#pragma unroll
    for (int k = 0; k < kRows; ++k) {
      const int r = q0 - (KT - 1) + k;
      const int rr = r < q0 + count ? r : q0 + count - 1;  // (rows behind the tile: the last one again, not used)
      input(rr, col, x[k]);
      if (two) input(rr, col + step, x2[k]);
    }
    float w[KT][V], w2[KT][V];
#pragma unroll
    for (int j = 0; j < KT; ++j) {
#pragma unroll
      for (int e = 0; e < V; ++e) w[j][e] = w2[j][e] = 1.f;
      if (a.taps) {
        get_floats<V>(a.taps + static_cast<size_t>(j) * channels + col, w[j]);
        if (two) get_floats<V>(a.taps + static_cast<size_t>(j) * channels + col + step, w2[j]);
      }
    }
    // whole tiles of values whose tokens lie side by side in a page: a store of eight tokens per channel
    const bool whole_run = sizeof(T) == 2 && TOK == 8 && role == kValue && count == 8 && (start + q0) % 8 == 0 &&
                           a.page_size % 8 == 0;
    uint32_t packed[V][TOK / 2 > 0 ? TOK / 2 : 1];
#pragma unroll
    for (int k = 0; k < TOK; ++k) {
      if (k >= count) break;
      float y[V], z[V];
#pragma unroll
      for (int e = 0; e < V; ++e) {
        y[e] = z[e] = 0.f;
#pragma unroll
        for (int j = 0; j < KT; ++j) {
          y[e] = fmaf(w[j][e], x[k + j][e], y[e]);
          if (two) z[e] = fmaf(w2[j][e], x2[k + j][e], z[e]);
        }
      }
      if (whole_run) {
#pragma unroll
        for (int e = 0; e < V; ++e) {
          const uint32_t bits = bf16_bits(y[e]);
          packed[e][k / 2] = k % 2 ? packed[e][k / 2] | (bits << 16) : bits;
        }
      } else {
        finish(k, y, z);
      }
    }
    if constexpr (TOK == 8 && sizeof(T) == 2) {
      if (whole_run) {
        const int pos = start + q0;
        const int page = a.tables[static_cast<size_t>(seq) * a.table_stride + pos / a.page_size];
        if (page >= 0 && page < a.num_pages) {
          T* dst = static_cast<T*>(a.v_pool) + (static_cast<size_t>(page) * a.v_heads * a.v_dim + i) * a.page_size +
                   pos % a.page_size;
#pragma unroll
          for (int e = 0; e < V; ++e)
            *reinterpret_cast<uint4*>(dst + static_cast<size_t>(e) * a.page_size) =
                make_uint4(packed[e][0], packed[e][1], packed[e][2], packed[e][3]);
        }
      }
    }
    if (KT > 1 && slot && q0 == 0) {
      // the last KT - 1 inputs: of the tile's own window where the portion ends in it, else of later rows
#pragma unroll
      for (int e = 0; e < KT - 1; ++e) {
        float keep[V], keep2[V];
        if (len <= TOK) {
#pragma unroll
          for (int k = 0; k < kRows; ++k)
            if (k == e + len) {
#pragma unroll
              for (int v = 0; v < V; ++v) keep[v] = x[k][v], keep2[v] = x2[k][v];
            }
        } else {
          input(len - (KT - 1) + e, col, keep);
          if (two) input(len - (KT - 1) + e, col + step, keep2);
        }
        float* dst = slot + static_cast<size_t>(e) * channels + col;
        put_run<float, V>(dst, keep);
        if (two) put_run<float, V>(dst + step, keep2);
      }
    }
  } else {
    const bool two = role == kTurned;
    for (int k = 0; k < count; ++k) {
      float y[V], z[V], x[V], w[V];
#pragma unroll
      for (int e = 0; e < V; ++e) y[e] = z[e] = 0.f;
      for (int j = 0; j < K; ++j) {
        input(q0 + k - (K - 1) + j, col, x);
        get_floats<V>(a.taps + static_cast<size_t>(j) * channels + col, w);
#pragma unroll
        for (int e = 0; e < V; ++e) y[e] = fmaf(w[e], x[e], y[e]);
        if (two) {
          input(q0 + k - (K - 1) + j, col + step, x);
          get_floats<V>(a.taps + static_cast<size_t>(j) * channels + col + step, w);
#pragma unroll
          for (int e = 0; e < V; ++e) z[e] = fmaf(w[e], x[e], z[e]);
        }
      }
      finish(k, y, z);
    }
    if (slot && q0 == 0) {
      for (int e = 0; e < K - 1; ++e) {  // ascending: entry e is read no more once it is written
        float keep[V];
        input(len - (K - 1) + e, col, keep);
        put_run<float, V>(slot + static_cast<size_t>(e) * channels + col, keep);
        if (two) {
          input(len - (K - 1) + e, col + step, keep);
          put_run<float, V>(slot + static_cast<size_t>(e) * channels + col + step, keep);
        }
      }
    }
  }
}

}  // namespace

}  // namespace shk

using namespace shk;

// Tokens of a portion that one workgroup takes.
extern "C" int shk_conv_store_tile(int taps) { return taps - 1 > kTile ? taps - 1 : kTile; }

extern "C" long long shk_conv_store_state_floats(int channels, int taps) {
  return static_cast<long long>(taps > 1 ? taps - 1 : 0) * channels;
}

extern "C" int shk_conv_store(const void* proj, int ldp, const float* parts, int splits, const float* bias, int dtype,
                              int n, const float* taps, int num_taps, int q_heads, int k_heads, int maps, int dim,
                              int rot_dim, const float* inv_freq, float magnitude, int v_heads, int v_dim, int gates,
                              const int32_t* positions, const int32_t* cu_q, const int32_t* slots,
                              const int32_t* tables, int table_stride, float* state, long long slot_stride,
                              const int32_t* tile_lists, int num_single, int num_tiles, void* q_out, float* gate_out,
                              void* k_pool, void* v_pool, int page_size, int num_pages, void* stream) {
  SHK_REQUIRE(dtype == kF32 || dtype == kBF16, "conv_store: unknown dtype %d", dtype);
  SHK_REQUIRE(n >= 0 && q_heads > 0 && k_heads >= 0 && maps > 0 && q_heads % maps == 0 && k_heads % maps == 0 && dim > 0 &&
                  v_heads >= 0 && gates >= 0 && (k_heads > 0) == (v_heads > 0) && (v_heads == 0 || v_dim > 0),
              "conv_store: bad sizes n=%d q_heads=%d k_heads=%d maps=%d dim=%d v_heads=%d v_dim=%d", n, q_heads, k_heads,
              maps, dim, v_heads, v_dim);
  SHK_REQUIRE(rot_dim >= 0 && rot_dim <= dim && rot_dim % 2 == 0 && rot_dim / 2 <= kMaxRotHalf,
              "conv_store: rot_dim %d must be even, at most dim %d and at most %d", rot_dim, dim, 2 * kMaxRotHalf);
  SHK_REQUIRE(num_taps >= 1 && num_taps <= kMaxTaps, "conv_store: %d taps are outside 1..%d", num_taps, kMaxTaps);
  const int channels = (q_heads + k_heads) * dim + v_heads * v_dim;
  SHK_REQUIRE(ldp >= channels + gates, "conv_store: rows of %d do not hold %d channels and %d gates", ldp, channels, gates);
  SHK_REQUIRE(splits >= 0 && (splits == 0 ? proj != nullptr : parts != nullptr), "conv_store: no projections");
  if (n == 0) return 0;
  SHK_REQUIRE(num_single >= 0 && num_tiles >= 0 && num_single + num_tiles > 0 && (num_tiles == 0 || tile_lists),
              "conv_store: no tiles");
  SHK_REQUIRE(positions && cu_q && slots && q_out && (rot_dim == 0 || inv_freq) && (gates == 0 || gate_out),
              "conv_store: null pointer");
  SHK_REQUIRE(num_taps == 1 || (taps && state && slot_stride >= shk_conv_store_state_floats(channels, num_taps)),
              "conv_store: a slot of %lld floats does not hold the convolution's inputs", slot_stride);
  if (k_heads)
    SHK_REQUIRE(tables && k_pool && v_pool && page_size > 0 && num_pages > 0 && table_stride > 0,
                "conv_store: bad cache (page_size=%d num_pages=%d table_stride=%d)", page_size, num_pages, table_stride);
  ConvStore a;
  a.proj = proj, a.ldp = ldp, a.parts = parts, a.splits = splits, a.part_stride = static_cast<size_t>(n) * ldp;
  a.bias = bias, a.taps = taps, a.K = num_taps;
  a.q_heads = q_heads, a.k_heads = k_heads, a.dim = dim, a.rot_dim = rot_dim, a.v_heads = v_heads, a.v_dim = v_dim;
  a.gates = gates, a.maps = maps, a.inv_freq = inv_freq, a.magnitude = magnitude;
  a.positions = positions, a.cu_q = cu_q, a.slots = slots, a.tables = tables, a.table_stride = table_stride;
  a.state = state, a.slot_stride = slot_stride, a.num_single = num_single;
  a.tile_seq = tile_lists, a.tile_q0 = tile_lists ? tile_lists + num_tiles : nullptr;
  a.tile = num_tiles ? shk_conv_store_tile(num_taps) : 1;
  a.q_out = q_out, a.gate_out = gate_out, a.k_pool = k_pool, a.v_pool = v_pool, a.page_size = page_size;
  a.num_pages = num_pages;
  bool four = dim % 4 == 0 && (rot_dim / 2) % 4 == 0 && (v_heads == 0 || v_dim % 4 == 0) && ldp % 4 == 0 && channels % 4 == 0 &&
              slot_stride % 4 == 0;
  for (const void* p : {proj, static_cast<const void*>(parts), static_cast<const void*>(taps),
                        static_cast<const void*>(state), static_cast<const void*>(q_out), static_cast<const void*>(k_pool),
                        static_cast<const void*>(v_pool)})
    four = four && reinterpret_cast<uintptr_t>(p) % 16 == 0;
  // few single tokens: a channel a thread, so that their launch has workgroups enough (the same sums either way)
  if (a.tile == 1 && static_cast<long long>(num_single) * (channels / 4) < 128 * kConvThreads) four = false;
  const int V = four ? 4 : 1;
  const int items = channels / V - (q_heads + k_heads) * (rot_dim / 2) / V + gates;
  const dim3 grid(num_single + num_tiles, (items + kConvThreads - 1) / kConvThreads);
  SHK_REQUIRE(grid.y <= 65535, "conv_store: too many channels");
  hipStream_t s = static_cast<hipStream_t>(stream);
  const size_t lds = static_cast<size_t>(a.tile) * rot_dim * sizeof(float);
  SHK_REQUIRE(lds <= 65536, "conv_store: the rotation's table does not fit a workgroup's LDS");
#define SHK_GO(T, V_, KT, TOK) conv_store_kernel<T, V_, KT, TOK><<<grid, kConvThreads, lds, s>>>(a)
#define SHK_TAPS(T, V_, TOK)                     \
  switch (num_taps) {                            \
    case 1: SHK_GO(T, V_, 1, TOK); break;        \
    case 2: SHK_GO(T, V_, 2, TOK); break;        \
    case 3: SHK_GO(T, V_, 3, TOK); break;        \
    case 4: SHK_GO(T, V_, 4, TOK); break;        \
    default: SHK_GO(T, V_, 0, TOK); break;       \
  }
#define SHK_TILE(T, V_)                          \
  do {                                           \
    if (a.tile == 1) SHK_TAPS(T, V_, 1)          \
    else SHK_TAPS(T, V_, kTile)                  \
  } while (0)
  if (dtype == kF32) {
    if (four) SHK_TILE(float, 4);
    else SHK_TILE(float, 1);
  } else {
    if (four) SHK_TILE(bf16, 4);
    else SHK_TILE(bf16, 1);
  }
#undef SHK_TILE
#undef SHK_TAPS
#undef SHK_GO
  SHK_LAUNCH_CHECK("conv_store");
  return 0;
}
