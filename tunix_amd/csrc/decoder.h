// Device helpers shared by the dense-weight decoder kernels (dense.hip, decoder_ops.hip,
// sink_attention.hip, lightning.hip): element access by dtype, activations, fragment order.
#pragma once
#include "common.h"

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

static inline bool src_given(const tnx_rows_src& s) { return s.ld > 0 && (s.split_k > 1 ? s.ws != nullptr : s.y != nullptr); }
