// Differential attention over the paged cache, general form.  A query head is `maps` attentions over
// the same values (two, or one: ordinary attention): map m scores its own query q[h, m] against its
// own keys k[g, m], and with two maps the head's result is
//   o = a1 - lambda a2,  o <- o / sqrt(mean(o^2) + eps) * (1 - diff)
// (the mean over the head's v_dim elements); either way it may be multiplied by one number per token
// and head, gate[t, h].  A window keeps a sequence's first tokens: the query at position i reads
// keys j <= i with i - j < window or j < keep_first.
//
// The key cache holds a key/value head's maps side by side as one row of maps * dim elements, queries
// likewise: q is [n, heads, maps * dim].
//
// diff_attention_kernel: one workgroup per (query token, query head), any sizes up to 256 elements a
// map and 256 a value, any page size, float32 or bfloat16 storage, float32 arithmetic.  A token's
// keys are walked in tiles of 256 counted from its own first key, so a token's result does not depend
// on how the step was cut.
#include "api.h"
#include "common.h"
#include "diff_mask.h"

namespace shk {

namespace {

constexpr int kDiffThreads = 256;
constexpr int kDiffMaxDim = 256;

template <typename T>
__global__ void __launch_bounds__(kDiffThreads)
    diff_attention_kernel(const T* __restrict__ q, T* __restrict__ out, int heads, int kv_heads, int maps, int dim,
                          int v_dim, const int32_t* __restrict__ positions, const int32_t* __restrict__ token_seq,
                          const int32_t* __restrict__ tables, int table_stride, const T* __restrict__ k_pool,
                          const T* __restrict__ v_pool, int page_size, int num_pages, int window, int keep_first,
                          float scale, float lambda, float rest, float eps, const float* __restrict__ gate) {
  __shared__ float qs[2 * kDiffMaxDim];
  __shared__ float probs[kDiffThreads];
  __shared__ int32_t rows[kDiffThreads];  // cache row of each key of the tile, -1 if there is none
  __shared__ float scratch[16];
  __shared__ float partial[kDiffThreads];
  __shared__ float result[2][kDiffMaxDim];
  const int head = blockIdx.x, t = blockIdx.y;
  const int g = head / (heads / kv_heads);
  const int pos = positions[t];
  const int32_t* table = tables + static_cast<size_t>(token_seq[t]) * table_stride;
  const int width = maps * dim, slab = key_slab(width);
  // the keys it reads: kept ones before its window, then the window's
  const int lo = first_key(pos, window, 0);
  const int kept = keep_first < lo ? keep_first : lo;
  const int total = kept + pos - lo + 1;

  const T* qrow = q + (static_cast<size_t>(t) * heads + head) * width;
  for (int d = threadIdx.x; d < width; d += kDiffThreads) qs[d] = to_float(qrow[d]);
  __syncthreads();
  const int groups = kDiffThreads / v_dim;  // threads (group, d) sum keys group, group + groups, ...
  const int group = threadIdx.x / v_dim, d = threadIdx.x % v_dim;
  const bool active = group < groups;

  for (int m = 0; m < maps; ++m) {
    float m_run = -INFINITY, l_run = 0.f, acc = 0.f;
    for (int x0 = 0; x0 < total; x0 += kDiffThreads) {
      const int x = x0 + threadIdx.x;
      float s = -INFINITY;
      int32_t row = -1;
      if (x < total) {
        const int j = x < kept ? x : lo + x - kept;
        const int page = table[j / page_size];
        if (page >= 0 && page < num_pages) {
          row = (page * kv_heads + g) * page_size + j % page_size;
          const T* head_keys = k_pool + static_cast<size_t>(page * kv_heads + g) * page_size * width;
          float dot = 0.f;
          if (slab == width) {  // the row in one piece
            const T* kr = head_keys + static_cast<size_t>(j % page_size) * width + m * dim;
            for (int e = 0; e < dim; ++e) dot = fmaf(qs[m * dim + e], to_float(kr[e]), dot);
          } else {
            for (int e = m * dim; e < (m + 1) * dim; ++e)
              dot = fmaf(qs[e], to_float(head_keys[(static_cast<size_t>(e / 32) * page_size + j % page_size) * 32 + e % 32]), dot);
          }
          s = dot * scale;
        }
      }
      const float m_new = fmaxf(m_run, block_max(s, scratch));
      const float p = row >= 0 ? expf(s - m_new) : 0.f;
      const float alpha = expf(m_run - m_new);  // 0 on the first tile
      probs[threadIdx.x] = p;
      rows[threadIdx.x] = row;
      const float tile_sum = block_sum(p, scratch);  // has the barriers that publish probs and rows
      l_run = l_run * alpha + tile_sum;
      m_run = m_new;
      if (active) {
        float a = 0.f;
        const int count = total - x0 < kDiffThreads ? total - x0 : kDiffThreads;
        for (int jj = group; jj < count; jj += groups) {
          const int32_t r = rows[jj];
          if (r < 0) continue;
          a = fmaf(probs[jj], to_float(v_pool[(static_cast<size_t>(r / page_size) * v_dim + d) * page_size + r % page_size]), a);
        }
        acc = acc * alpha + a;
      }
      __syncthreads();  // probs and rows are rewritten by the next tile
    }
    partial[threadIdx.x] = active ? acc : 0.f;
    __syncthreads();
    if (threadIdx.x < v_dim) {
      float sum = 0.f;
      for (int gg = 0; gg < groups; ++gg) sum += partial[gg * v_dim + threadIdx.x];
      result[m][threadIdx.x] = sum / l_run;
    }
    __syncthreads();
  }
  float o = 0.f;
  const bool mine = threadIdx.x < v_dim;
  if (mine) o = maps == 2 ? result[0][threadIdx.x] - lambda * result[1][threadIdx.x] : result[0][threadIdx.x];
  if (maps == 2) {
    const float ss = block_sum(o * o, scratch);
    o = o / sqrtf(ss / static_cast<float>(v_dim) + eps) * rest;
  }
  if (gate) o *= gate[static_cast<size_t>(t) * heads + head];
  if (mine) out[(static_cast<size_t>(t) * heads + head) * v_dim + threadIdx.x] = from_float<T>(o);
}

}  // namespace

}  // namespace shk

using namespace shk;

extern "C" int shk_diff_attention(const void* q, void* out, int dtype, int n, int heads, int kv_heads, int maps, int dim,
                                  int v_dim, const int32_t* positions, const int32_t* token_seq, const int32_t* tables,
                                  int table_stride, int num_seqs, const void* k_pool, const void* v_pool, int page_size,
                                  int num_pages, int window, int keep_first, float scale, float lambda, float rest,
                                  float eps, const float* gate, void* stream) {
  SHK_REQUIRE(dtype == kF32 || dtype == kBF16, "diff_attention: unknown dtype %d", dtype);
  SHK_REQUIRE(n >= 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0,
              "diff_attention: heads=%d must be a positive multiple of kv_heads=%d", heads, kv_heads);
  SHK_REQUIRE(maps == 1 || maps == 2, "diff_attention: %d maps a head (1 or 2)", maps);
  SHK_REQUIRE(dim > 0 && dim <= kDiffMaxDim && v_dim > 0 && v_dim <= kDiffThreads,
              "diff_attention: sizes dim=%d v_dim=%d are outside 1..256", dim, v_dim);
  SHK_REQUIRE(window >= 0 && keep_first >= 0, "diff_attention: bad mask window=%d keep_first=%d", window, keep_first);
  SHK_REQUIRE(page_size > 0 && num_pages > 0 && table_stride > 0 && num_seqs > 0,
              "diff_attention: bad cache sizes page_size=%d num_pages=%d table_stride=%d num_seqs=%d", page_size, num_pages,
              table_stride, num_seqs);
  SHK_REQUIRE(static_cast<int64_t>(num_pages) * kv_heads * page_size < (1LL << 31),
              "diff_attention: cache pool has too many rows for 32-bit row indices");
  if (n == 0) return 0;
  SHK_REQUIRE(n <= 65535, "diff_attention: at most 65535 tokens a call, got %d", n);
  SHK_REQUIRE(q && out && positions && token_seq && tables && k_pool && v_pool, "diff_attention: null pointer");
  hipStream_t s = static_cast<hipStream_t>(stream);
  const dim3 grid(heads, n);
#define SHK_GO(T)                                                                                                  \
  diff_attention_kernel<T><<<grid, kDiffThreads, 0, s>>>(                                                          \
      static_cast<const T*>(q), static_cast<T*>(out), heads, kv_heads, maps, dim, v_dim, positions, token_seq,     \
      tables, table_stride, static_cast<const T*>(k_pool), static_cast<const T*>(v_pool), page_size, num_pages,    \
      window, keep_first, scale, lambda, rest, eps, gate)
  if (dtype == kF32) SHK_GO(float);
  else SHK_GO(bf16);
#undef SHK_GO
  SHK_LAUNCH_CHECK("diff_attention");
  return 0;
}
