// Device helpers shared by the dense-weight decoder kernels (dense.hip, decoder_ops.hip,
// sink_attention.hip, lightning.hip, ssd.hip, latent.hip, memory.hip, mixed_attention.hip, layer_ops.hip,
// gated_state.hip): element access by dtype, activations,
// fragment order, MFMA.
#pragma once
#include "common.h"

typedef float f32x16 __attribute__((ext_vector_type(16)));
__device__ __forceinline__ f32x16 mfma32(u32x4 a, u32x4 b, f32x16 c) {
  // D[32x32] += A[32x16] * B[16x32]; lane l holds A row l%32 / B column l%32, k = 8*(l/32)..+7;
  // D: column l%32, rows 8*(r/4) + 4*(l/32) + r%4 for register r.
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}
// bf16 pairs of (x, y) and of what that rounding left out: together 16 mantissa bits
__device__ __forceinline__ void split2(float x, float y, uint32_t& hi, uint32_t& lo) {
  hi = cvt_pk_bf16(x, y);
  lo = cvt_pk_bf16(x - bflo(hi), y - bfhi(hi));
}

__device__ __forceinline__ float gelu_tanh_f32(float z) {
  const float k0 = 0.7978845608028654f, k1 = 0.044715f;
  return 0.5f * z * (1.0f + tanhf(k0 * (z + k1 * z * z * z)));
}
__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f32(float z) { return z / (1.0f + expf(-z)); }

// T = uint16_t (bf16 bits) or float
__device__ __forceinline__ float ld_elem(const uint16_t* p, int64_t i) { return bf2f(p[i]); }
__device__ __forceinline__ float ld_elem(const float* p, int64_t i) { return p[i]; }
__device__ __forceinline__ void st_elem(uint16_t* p, int64_t i, float v) { p[i] = f2bf(v); }
__device__ __forceinline__ void st_elem(float* p, int64_t i, float v) { p[i] = v; }

// Fragment order of a [M, K] bf16 activation matrix (K a multiple of 16): blocks of 32 rows x 16 k,
// k fastest over the blocks, inside a block the B operand of a 32x32x16 MFMA: lane l holds row
// l % 32, k = 8 (l / 32) .. + 7.  A wave reads a block as one contiguous kilobyte.  Runs of eight
// consecutive k (from a multiple of eight) stay contiguous.
__host__ __device__ __forceinline__ int64_t frag_index(int64_t m, int64_t k, int64_t K) {
  return (((m >> 5) * (K >> 4) + (k >> 4)) << 9) + (((k >> 3) & 1) << 8) + ((m & 31) << 3) + (k & 7);
}

// A linear's output row: finished values (T) or the fp32 partial planes of a k-split linear, which
// the reader sums in split order.  `plane` is the distance between planes in elements.
template <typename T>
struct RowSrc {
  const T* y;
  const float* ws;
  int split;
  int64_t plane, ld;
  __device__ __forceinline__ float get(int64_t row, int64_t col) const {
    const int64_t o = row * ld + col;
    if (split <= 1) return ld_elem(y, o);
    float v = 0.f;
    for (int z = 0; z < split; ++z) v += ws[z * plane + o];
    return v;
  }
};

// Eight consecutive values of a row (col, ld and planes on 8-element boundaries); partial planes are
// requested together, four at a time, and added in plane order.
template <typename T>
__device__ __forceinline__ void get8(const RowSrc<T>& s, int64_t row, int64_t col, float (&f)[8]) {
  const int64_t o = row * s.ld + col;
  if (s.split > 1) {
    const float* p = s.ws + o;
#pragma unroll
    for (int j = 0; j < 8; ++j) f[j] = 0.f;
    for (int z0 = 0; z0 < s.split; z0 += 4) {
      f32x4 a[4], b[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const float* q = p + (int64_t)min(z0 + u, s.split - 1) * s.plane;
        a[u] = *reinterpret_cast<const f32x4*>(q);
        b[u] = *reinterpret_cast<const f32x4*>(q + 4);
      }
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (z0 + u < s.split)
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            f[j] += a[u][j];
            f[4 + j] += b[u][j];
          }
    }
  } else if constexpr (sizeof(T) == 2) {
    const u32x4 v = *reinterpret_cast<const u32x4*>(s.y + o);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      f[2 * j] = bflo(v[j]);
      f[2 * j + 1] = bfhi(v[j]);
    }
  } else {
    const f32x4 a = *reinterpret_cast<const f32x4*>(s.y + o), b = *reinterpret_cast<const f32x4*>(s.y + o + 4);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      f[j] = a[j];
      f[4 + j] = b[j];
    }
  }
}
__device__ __forceinline__ void put8(uint16_t* p, const float (&f)[8]) {
  *reinterpret_cast<u32x4*>(p) = u32x4{pack2bf(f[0], f[1]), pack2bf(f[2], f[3]), pack2bf(f[4], f[5]), pack2bf(f[6], f[7])};
}
__device__ __forceinline__ void put8(float* p, const float (&f)[8]) {
  *reinterpret_cast<f32x4*>(p) = f32x4{f[0], f[1], f[2], f[3]};
  *reinterpret_cast<f32x4*>(p + 4) = f32x4{f[4], f[5], f[6], f[7]};
}

static inline bool src_given(const tnx_rows_src& s) { return s.ld > 0 && (s.split_k > 1 ? s.ws != nullptr : s.y != nullptr); }
