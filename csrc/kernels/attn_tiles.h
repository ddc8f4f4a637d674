// Shared by the attention kernels that stage cache rows in LDS as they are (prompt_attention.hip, split_attention.hip): rows of
// 16-byte chunks, chunk c of row r stored at c ^ swz(r), read as MFMA fragments along the row (keys) or, through the LDS
// transpose read, down the rows (values).
#pragma once
#include "common.h"
#include "direct_lds.h"

constexpr float ATT_LOG2E = 1.44269504088896341f;

typedef short s16x4 __attribute__((ext_vector_type(4)));

// transpose read: the 16 lanes of a group hand in 8-byte pieces of a 4 x 16 matrix (lane l: row l / 4, columns 4 (l % 4) ..);
// lane i receives column i
SYM_DEV uint2 read_tr(const char* lds) {
  const s16x4 v = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)lds);
  return __builtin_bit_cast(uint2, v);
}

// 16-byte chunks per LDS row of a head of D entries (a power of two), and the row's XOR
constexpr int row_chunks(int D) { return D <= 32 ? 4 : (D <= 64 ? 8 : 16); }
template <int CH>
SYM_DEV int swz(int r) {
  if constexpr (CH == 16) return 4 * (r & 3) + ((r >> 2) & 3);
  else if constexpr (CH == 8) return 4 * ((r >> 1) & 1) + ((r >> 2) & 3);
  else return (r >> 2) & 3;
}

// cache row of position kp of a sequence (block table bt): a shift and a mask for power-of-two blocks
SYM_DEV long long cache_row(const int* __restrict__ bt, int kp, int BS, int shift) {
  return shift >= 0 ? ((long long)bt[kp >> shift] << shift) + (kp & (BS - 1)) : (long long)bt[kp / BS] * BS + kp % BS;
}
