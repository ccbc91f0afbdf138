// LDS tile helpers shared by the attention kernels (attn.hip, xattn_mfma.hip).
#pragma once
#include "md_common.h"

constexpr int kVSub = 1056;  // bytes per [32 keys][16 d] V sub-tile (+32 B pad: conflict-free ds_write_b128)

__device__ __forceinline__ bf16x8 lds_read_b128(const unsigned char* p) {
    return *reinterpret_cast<const bf16x8*>(p);
}
__device__ __forceinline__ bf16x4 lds_read_tr(const unsigned char* p) {
    return __builtin_amdgcn_ds_read_tr16_b64_v4bf16(
        (__attribute__((address_space(3))) bf16x4*)(p));
}
