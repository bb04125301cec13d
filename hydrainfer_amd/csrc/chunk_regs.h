// chunk_regs.h — a chunk of tokens of one operand of a recurrence on its way from global memory to LDS.
#pragma once
#include "hx_common.h"

namespace hx {

// One operand's chunk [TC tokens][KP channels] on its way from global memory (rows of `dtype`, K valid channels) to LDS (rows
// STRIDE floats apart): thread `tid` of 256 holds NI groups of four channels AS THEY CAME (float bits, or four bfloat16 in two words).  Nothing is
// computed on them before store(): the scan between fetch() and store() then waits for no load.
template <int TC, int KP, int STRIDE = KP>
struct ChunkRegs {
  static constexpr int kGroups = TC * KP / 4;
  static constexpr int NI = (kGroups + 255) / 256;
  u32x4 r[NI];

  __device__ __forceinline__ void fetch(const void* base, int dtype, int64_t stride, int64_t first_elem, int K, int64_t t0, int n_tok,
                                        bool by4, int tid) {
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int g = tid + i * 256;
      const int row = g / (KP / 4), c = (g % (KP / 4)) * 4;
      u32x4 v = u32x4{0u, 0u, 0u, 0u};
      if (g < kGroups && row < n_tok && c < K) {
        const int64_t e = (t0 + row) * stride + first_elem + c;
        if (by4 && c + 3 < K) {
          if (dtype == HX_F32) {
            v = *reinterpret_cast<const u32x4*>((const float*)base + e);
          } else {
            const u32x2 b = *reinterpret_cast<const u32x2*>((const u16*)base + e);
            v[0] = b[0];
            v[1] = b[1];
          }
        } else if (dtype == HX_F32) {
#pragma unroll
          for (int j = 0; j < 4; ++j)
            if (c + j < K) v[j] = ((const uint32_t*)base)[e + j];
        } else {
#pragma unroll
          for (int j = 0; j < 4; ++j)
            if (c + j < K) v[j >> 1] |= (uint32_t)((const u16*)base)[e + j] << (16 * (j & 1));
        }
      }
      r[i] = v;
    }
  }

  // fn: what happens to every element on its way
  template <typename F>
  __device__ __forceinline__ void store(float* lds, int dtype, int tid, F fn) const {
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int g = tid + i * 256;
      if (g < kGroups) {
        u32x4 v = r[i];
        if (dtype != HX_F32) v = u32x4{v[0] << 16, v[0] & 0xffff0000u, v[1] << 16, v[1] & 0xffff0000u};
        f32x4 f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const uint32_t bits = v[j];      // (a copy: a bit cast of a vector's element in place takes the vector's first)
          f[j] = fn(__builtin_bit_cast(float, bits));
        }
        *reinterpret_cast<f32x4*>(lds + (STRIDE == KP ? 4 * g : (g / (KP / 4)) * STRIDE + (g % (KP / 4)) * 4)) = f;
      }
    }
  }
  __device__ __forceinline__ void store(float* lds, int dtype, int tid) const {
    store(lds, dtype, tid, [](float x) { return x; });
  }
};

}  // namespace hx
