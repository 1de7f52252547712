// What the attention kernels of hybrid decoders share.
#pragma once

#include <atomic>

#include "common.h"

namespace {

typedef __bf16 la_v4bf __attribute__((__vector_size__(4 * sizeof(__bf16))));
typedef __attribute__((address_space(3))) la_v4bf la_lds_v4bf;
typedef uint32_t la_u2 __attribute__((ext_vector_type(2)));
typedef uint32_t la_u4 __attribute__((ext_vector_type(4)));

constexpr float LOG2E = 1.4426950408889634f;

// 8 elements of one column of a row-major LDS tile: 4 rows from `p`, 4 from `p2` (see the
// transposing read's lane layout in attention_prefill.hip)
__device__ __forceinline__ bf16x8_t read_column8(const char* p, const char* p2) {
  const la_u2 lo = __builtin_bit_cast(la_u2, __builtin_amdgcn_ds_read_tr16_b64_v4bf16((la_lds_v4bf*)p));
  const la_u2 hi = __builtin_bit_cast(la_u2, __builtin_amdgcn_ds_read_tr16_b64_v4bf16((la_lds_v4bf*)p2));
  const la_u4 w = {lo[0], lo[1], hi[0], hi[1]};
  return __builtin_bit_cast(bf16x8_t, w);
}

// allows a kernel that much dynamic LDS, once per device (`done`: one bit each)
bool raise_lds(const void* kernel, int bytes, std::atomic<uint64_t>& done) {
  int dev = 0;
  if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) return false;
  const uint64_t bit = 1ull << dev;
  if (done.load(std::memory_order_acquire) & bit) return true;
  if (hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, bytes) != hipSuccess)
    return false;
  done.fetch_or(bit, std::memory_order_release);
  return true;
}

// keys of one split
__device__ __forceinline__ int split_keys(int n_keys, int splits) {
  return ((n_keys + splits - 1) / splits + 15) & ~15;
}

}  // namespace
