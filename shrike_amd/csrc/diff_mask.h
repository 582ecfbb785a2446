// Which keys a query reads under a window that keeps a sequence's first tokens, and how the kernels on
// the matrix units walk them in chunks of 32: the chunks that hold kept keys, then those from the one
// with the window's first key on, none twice.
#pragma once

#include "common.h"

namespace shk {

// The query at `pos`, whose window's first key is `lo`, reads key j.
__device__ __forceinline__ bool reads_key(int j, int pos, int lo, int keep_first) {
  return j <= pos && (j >= lo || j < keep_first);
}

// The chunks of a run of queries whose windows begin at `lo` or later: chunk c starts at key_of(c).
struct KeptChunks {
  int kept;   // chunks of kept keys before the window's first chunk
  int first;  // the window's first chunk starts here
  __device__ __forceinline__ KeptChunks(int lo, int keep_first) {
    first = lo & ~31;
    const int want = (keep_first + 31) / 32;
    kept = want < first / 32 ? want : first / 32;
  }
  __device__ __forceinline__ int count(int pos_max) const { return kept + (pos_max - first) / 32 + 1; }
  __device__ __forceinline__ int key_of(int c) const { return c < kept ? 32 * c : first + 32 * (c - kept); }
};

// A key whose page the sequence holds, for a load that begins at `key`: the key itself where some query
// of the run reads it or it lies in a kept page, else the nearest key that is read.
__device__ __forceinline__ int held_key(int key, int pos_max, int lo, int keep_first) {
  const int k = (key < keep_first || key >= lo) ? key : lo;
  return k > pos_max ? pos_max : k;
}

}  // namespace shk
