// Causal grouped-query attention with a learned sink per head, separate key and value head sizes
// and an arbitrary score scale, over caches K [B, G, S, dkp] and V [B, G, S, dvp] whose rows are
// zero-padded.  Scores, softmax and its running sums are fp32.  A row's keys start at starts[b]
// (left padding), whatever their token ids.  A head may take off its score a slope times the distance, and a position may
// see its own chunk of positions only (BIAS).
//
//   sink_attn_tile_kernel   many query positions: 128 query rows per work-group, keys and values
//                           staged through LDS, 32x32x16 MFMAs
//   sink_attn_step_kernel   few query rows (decode): one wave per 16 query rows and key chunk,
//                           keys and values streamed through registers, 16x16x32 MFMAs
//   sink_attn_any_kernel    any sizes and fp32: plain loops
#include <string.h>

#include "decoder.h"

namespace {

struct SinkArgs {
  int64_t B, T, S;
  int H, G, R, dk, dv, dkp, dvp;
  float scale;
  const void* q;
  const void* k;
  const void* v;
  const float* sinks;      // [H] or null
  const int32_t* starts;   // [B]
  const int32_t* col_ptr;
  int kv_chunk, n_chunks;
  float* ws;
  void* out;
  int64_t out_ld;
  int out_frag;
  int64_t out_head;        // distance of two heads in an output row
  const float* slopes;     // [H] or null
  int chunk;               // positions of a chunk, 0: no chunks
};

// the first column that the position in column `col` sees
__device__ __forceinline__ int first_seen(int col, int start, int chunk) {
  return chunk > 0 && col > start ? start + (col - start) / chunk * chunk : start;
}

constexpr float kNegBig = -1.0e30f;
constexpr float kLog2e = 1.4426950408889634f;
__device__ __forceinline__ float exp2_hw(float x) { return __builtin_amdgcn_exp2f(x); }

// Weight of the finished sum: O * result is the output.  m is in log2 units.
__device__ __forceinline__ float finish_scale(float m, float l, bool has_sink, float sink) {
  if (!has_sink) return l > 0.f ? 1.0f / l : 0.f;
  const float s2 = sink * kLog2e, top = fmaxf(m, s2);
  const float w = exp2_hw(m - top);
  return w / (l * w + exp2_hw(s2 - top));
}

// ---- any sizes ----------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void sink_attn_any_kernel(const SinkArgs a) {
  __shared__ float p[256], red[4];
  const int h = blockIdx.x, g = h / a.R;
  const int64_t row = blockIdx.y, b = row / a.T, t = row % a.T;
  const int tid = threadIdx.x, last = *a.col_ptr + (int)t, first = first_seen(last, a.starts[b], a.chunk);
  const float slope = a.slopes ? a.slopes[h] : 0.f;
  const T* q = reinterpret_cast<const T*>(a.q) + (row * a.H + h) * a.dkp;
  const T* k = reinterpret_cast<const T*>(a.k) + (b * a.G + g) * a.S * a.dkp;
  const T* v = reinterpret_cast<const T*>(a.v) + (b * a.G + g) * a.S * a.dvp;
  constexpr int kMaxOut = 8;   // dv <= 2048
  float o[kMaxOut] = {};
  float m = kNegBig, l = 0.f;
  if (last < a.S)
    for (int k0 = first; k0 <= last; k0 += 256) {
      const int key = k0 + tid, n = min(256, last - k0 + 1);
      float s = kNegBig;
      if (tid < n) {
        float d = 0.f;
        for (int i = 0; i < a.dk; ++i) d += ld_elem(q, i) * ld_elem(k, (int64_t)key * a.dkp + i);
        s = (d * a.scale - slope * (float)(last - key)) * kLog2e;
      }
      float mx = wave_max(s);
      __syncthreads();
      if ((tid & 63) == 0) red[tid >> 6] = mx;
      __syncthreads();
      mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
      const float mn = fmaxf(m, mx), alpha = exp2f(m - mn);
      m = mn;
      const float e = tid < n ? exp2f(s - mn) : 0.f;
      p[tid] = e;
      float sum = wave_sum(e);
      __syncthreads();
      if ((tid & 63) == 0) red[tid >> 6] = sum;
      __syncthreads();
      l = l * alpha + red[0] + red[1] + red[2] + red[3];
#pragma unroll
      for (int c = 0; c < kMaxOut; ++c) {
        const int d = c * 256 + tid;
        if (d >= a.dv) break;
        float acc = o[c] * alpha;
        for (int j = 0; j < n; ++j) acc += p[j] * ld_elem(v, (int64_t)(k0 + j) * a.dvp + d);
        o[c] = acc;
      }
    }
  float w;
  if (a.sinks) {
    const float s2 = a.sinks[h] * kLog2e, top = fmaxf(m, s2);
    const float e = exp2f(m - top);
    w = e / (l * e + exp2f(s2 - top));
  } else {
    w = l > 0.f ? 1.0f / l : 0.f;
  }
  T* out = reinterpret_cast<T*>(a.out);
#pragma unroll
  for (int c = 0; c < kMaxOut; ++c) {
    const int d = c * 256 + tid;
    if (d >= a.dv) break;
    const int64_t col = (int64_t)h * a.out_head + d;
    st_elem(out, a.out_frag ? frag_index(row, col, a.out_ld) : row * a.out_ld + col, o[c] * w);
  }
}

// ---- few query rows -----------------------------------------------------------------------------
// One wave per (16 query rows of a (row, kv head), key chunk).  S^T = K . q^T leaves every lane with
// the scores of one query for eight keys: the A fragment of the P . V product.  Keys and values flow
// through a ring of register stages; every load is unconditional so the waits count exactly.
template <int KS, int NH, int NJ, bool BIAS>   // 32-deep k-steps, halves of V, value columns per lane and half
__global__ __launch_bounds__(64) __attribute__((amdgpu_waves_per_eu(1, 2))) void sink_attn_step_kernel(const SinkArgs a) {
  constexpr int DK = KS * 32, DV = NH * NJ * 16;
  constexpr int NS = KS * 8 + NH * 4 * NJ <= 64 ? 2 : 1;
  typedef uint32_t vfrag __attribute__((ext_vector_type(NJ / 2)));
  const int lane = threadIdx.x, lm = lane & 15, lq = lane >> 4;
  const int chunk = blockIdx.x;
  const unsigned rows = (unsigned)(a.T * a.R), qts = (rows + 15) / 16;
  const int g = blockIdx.y / qts, qt = blockIdx.y % qts;
  const int64_t b = blockIdx.z;
  const int col0 = *a.col_ptr, start = a.starts[b];
  const unsigned qrow = (unsigned)qt * 16 + lm;
  const bool qvalid = qrow < rows;
  const int tq = qvalid ? (int)(qrow / a.R) : 0, rq = qvalid ? (int)(qrow % a.R) : 0;
  const int c_n = min(col0 + tq, (int)a.S - 1);
  const uint16_t* q = reinterpret_cast<const uint16_t*>(a.q) + ((b * a.T + tq) * a.H + g * a.R + rq) * DK;
  int k_lo = start, k_hi = min(col0 + (int)a.T - 1, (int)a.S - 1), split0 = 0, seen = start;
  float slope2 = 0.f;
  if constexpr (BIAS) {
    k_lo = first_seen(col0 + (int)(qt * 16u / a.R), start, a.chunk);   // (of the tile's first position; later ones see no earlier key)
    seen = first_seen(c_n, start, a.chunk);
    split0 = a.chunk > 0 ? first_seen(col0, start, a.chunk) & ~31 : 0;
    if (a.slopes) slope2 = a.slopes[g * a.R + rq] * kLog2e;
  }
  if (a.n_chunks > 1) {
    k_lo = max(k_lo, split0 + chunk * a.kv_chunk);
    k_hi = min(k_hi, split0 + chunk * a.kv_chunk + a.kv_chunk - 1);
  }
  u32x4 qf[KS];
#pragma unroll
  for (int j = 0; j < KS; ++j) qf[j] = qvalid ? *reinterpret_cast<const u32x4*>(q + j * 32 + lq * 8) : u32x4{0, 0, 0, 0};
  f32x4 O[NH][NJ];
#pragma unroll
  for (int h = 0; h < NH; ++h)
#pragma unroll
    for (int j = 0; j < NJ; ++j) O[h][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = kNegBig, l_run = 0.f;
  const uint32_t slab_k = (uint32_t)a.S * DK * 2u, slab_v = (uint32_t)a.S * DV * 2u;
  const rsrc_t rk = make_rsrc(reinterpret_cast<const uint16_t*>(a.k) + (b * a.G + g) * a.S * DK, slab_k);
  const rsrc_t rv = make_rsrc(reinterpret_cast<const uint16_t*>(a.v) + (b * a.G + g) * a.S * DV, slab_v);
  struct Stage {
    u32x4 kf[2][KS];
    vfrag vf[NH][8];
  };
  const uint32_t koff = (uint32_t)(lm * DK + lq * 8) * 2u, voff = (uint32_t)(4 * lq * DV + NJ * lm) * 2u;
  auto load_block = [&](int kb, Stage& sg) {
#pragma unroll
    for (int tt = 0; tt < 2; ++tt)
#pragma unroll
      for (int j = 0; j < KS; ++j)
        sg.kf[tt][j] = __builtin_amdgcn_raw_buffer_load_b128(rk, koff + (uint32_t)((kb + tt * 16) * DK * 2 + j * 64), 0, kStreamOnce);
#pragma unroll
    for (int s = 0; s < 8; ++s)
#pragma unroll
      for (int h = 0; h < NH; ++h) {
        const uint32_t o = voff + (uint32_t)((kb + (s < 4 ? s : 12 + s)) * DV * 2 + h * (NJ * 32));
        if constexpr (NJ == 8) sg.vf[h][s] = __builtin_amdgcn_raw_buffer_load_b128(rv, o, 0, kStreamOnce);
        else sg.vf[h][s] = __builtin_amdgcn_raw_buffer_load_b64(rv, o, 0, kStreamOnce);
      }
  };
  const float sc2 = a.scale * kLog2e;
  auto compute_block = [&](int kb, const Stage& sg) {
    f32x4 st[2];
#pragma unroll
    for (int tt = 0; tt < 2; ++tt) {
      st[tt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < KS; ++j) st[tt] = mfma16(sg.kf[tt][j], qf[j], st[tt]);
    }
    float sv[8], bmax = kNegBig;
    bool ok[8];
#pragma unroll
    for (int s = 0; s < 8; ++s) {
      const int key = kb + (s < 4 ? 4 * lq + s : 16 + 4 * lq + (s - 4));
      ok[s] = qvalid && key >= k_lo && key <= min(k_hi, c_n);
      if constexpr (BIAS) ok[s] = ok[s] && key >= seen;
      sv[s] = st[s >> 2][s & 3] * sc2;
      if constexpr (BIAS) sv[s] = __builtin_fmaf(slope2, (float)(key - c_n), sv[s]);
      if (ok[s]) bmax = fmaxf(bmax, sv[s]);
    }
    bmax = fmaxf(bmax, __shfl_xor(bmax, 16, 64));
    bmax = fmaxf(bmax, __shfl_xor(bmax, 32, 64));
    const float m_new = fmaxf(m_run, bmax), alpha = exp2_hw(m_run - m_new);
    m_run = m_new;
    float p[8], psum = 0.f;
#pragma unroll
    for (int s = 0; s < 8; ++s) {
      p[s] = ok[s] ? exp2_hw(sv[s] - m_new) : 0.f;
      psum += p[s];
    }
    l_run = l_run * alpha + psum;
    const u32x4 pa = {pack2bf(p[0], p[1]), pack2bf(p[2], p[3]), pack2bf(p[4], p[5]), pack2bf(p[6], p[7])};
    if (__builtin_amdgcn_ballot_w64(alpha != 1.0f) != 0) {
      float ar[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) ar[i] = __shfl(alpha, 4 * lq + i, 64);
#pragma unroll
      for (int h = 0; h < NH; ++h)
#pragma unroll
        for (int j = 0; j < NJ; ++j)
#pragma unroll
          for (int i = 0; i < 4; ++i) O[h][j][i] *= ar[i];
    }
#pragma unroll
    for (int h = 0; h < NH; ++h)
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        const uint32_t sel = (j & 1) ? 0x07060302u : 0x05040100u;
        u32x4 bf;
#pragma unroll
        for (int r = 0; r < 4; ++r) bf[r] = __builtin_amdgcn_perm(sg.vf[h][2 * r + 1][j >> 1], sg.vf[h][2 * r][j >> 1], sel);
        O[h][j] = mfma16(pa, bf, O[h][j]);
      }
  };
  if (k_lo <= k_hi) {
    Stage sg[NS];
    const int kb0 = k_lo & ~31, kb_last = k_hi & ~31;
    if constexpr (NS == 2) {
      load_block(kb0, sg[0]);
      for (int kb = kb0; kb <= kb_last; kb += 64) {
        load_block(min(kb + 32, kb_last), sg[1]);
        compute_block(kb, sg[0]);
        load_block(min(kb + 64, kb_last), sg[0]);
        if (kb + 32 <= kb_last) compute_block(kb + 32, sg[1]);
      }
    } else {
      for (int kb = kb0; kb <= kb_last; kb += 32) {
        load_block(kb, sg[0]);
        compute_block(kb, sg[0]);
      }
    }
  }
  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  // lane: queries 4 lq + i (i = 0..3), value columns h * 16 NJ + NJ lm + j
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float m = __shfl(m_run, 4 * lq + i, 64), l = __shfl(l_run, 4 * lq + i, 64);
    const unsigned qr = (unsigned)qt * 16 + 4 * lq + i;
    if (qr >= rows) continue;
    const int t = (int)(qr / a.R), r = (int)(qr % a.R), head = g * a.R + r;
    const int64_t row = b * a.T + t, qv = row * a.H + head;
    if (a.n_chunks > 1) {
      const int64_t nq = a.B * a.T * a.H;
      float* po = a.ws + (qv * a.n_chunks + chunk) * DV;
#pragma unroll
      for (int h = 0; h < NH; ++h)
#pragma unroll
        for (int j = 0; j < NJ; j += 4)
          *reinterpret_cast<f32x4*>(po + h * 16 * NJ + NJ * lm + j) = f32x4{O[h][j][i], O[h][j + 1][i], O[h][j + 2][i], O[h][j + 3][i]};
      if (lm == 0) {
        float* ml = a.ws + nq * a.n_chunks * DV + (qv * a.n_chunks + chunk) * 2;
        ml[0] = m;
        ml[1] = l;
      }
      continue;
    }
    const float w = finish_scale(m, l, a.sinks != nullptr, a.sinks ? a.sinks[head] : 0.f);
    uint16_t* out = reinterpret_cast<uint16_t*>(a.out);
#pragma unroll
    for (int h = 0; h < NH; ++h) {
      const int d0 = h * 16 * NJ + NJ * lm;
#pragma unroll
      for (int j = 0; j < NJ; ++j)
        if (d0 + j < a.dv) {
          const int64_t col = (int64_t)head * a.out_head + d0 + j;
          out[a.out_frag ? frag_index(row, col, a.out_ld) : row * a.out_ld + col] = f2bf(O[h][j][i] * w);
        }
    }
  }
}

// one work-group per query vector: merges the chunks and adds the sink
__global__ __launch_bounds__(128) void sink_attn_merge_kernel(const SinkArgs a) {
  extern __shared__ float wts[];   // [n_chunks]
  __shared__ float tot;
  const int64_t qv = blockIdx.x, row = qv / a.H;
  const int head = (int)(qv % a.H);
  const float* ml = a.ws + a.B * a.T * a.H * a.n_chunks * a.dvp + qv * a.n_chunks * 2;
  if (threadIdx.x < 64) {
    float m = kNegBig;
    for (int c = threadIdx.x; c < a.n_chunks; c += 64) m = fmaxf(m, ml[2 * c]);
    m = wave_max(m);
    float l = 0.f;
    for (int c = threadIdx.x; c < a.n_chunks; c += 64) {
      const float w = exp2_hw(ml[2 * c] - m);
      wts[c] = w;
      l += w * ml[2 * c + 1];
    }
    l = wave_sum(l);
    if (threadIdx.x == 0) tot = finish_scale(m, l, a.sinks != nullptr, a.sinks ? a.sinks[head] : 0.f);
  }
  __syncthreads();
  const float* po = a.ws + qv * a.n_chunks * a.dvp;
  uint16_t* out = reinterpret_cast<uint16_t*>(a.out);
  for (int d = threadIdx.x; d < a.dv; d += 128) {
    float acc = 0.f;
    for (int c = 0; c < a.n_chunks; ++c) acc += wts[c] * po[(int64_t)c * a.dvp + d];
    const int64_t col = (int64_t)head * a.out_head + d;
    out[a.out_frag ? frag_index(row, col, a.out_ld) : row * a.out_ld + col] = f2bf(acc * tot);
  }
}

// ---- many query rows ----------------------------------------------------------------------------
// Query rows of a (row, kv head) are (position, head of the group) pairs, heads fastest, so the heads
// that share keys share the staged tile.  A wave owns 32 of them.  Both products are formed
// transposed, S^T = K . Q^T and O^T = V^T . P^T: a lane holds the scores, the probabilities (already
// the B operand of the second product, in a permuted key order that the V fragments follow) and the
// output of ONE query, so the softmax state is per lane.
template <int KD, int NV, bool BIAS>   // 16-deep k-steps of the head size; 32-column groups of the value size
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(KD + NV > 11 ? 1 : 2, 2)))
void sink_attn_tile_kernel(const SinkArgs a) {
  constexpr int DK = KD * 16, DV = NV * 32, KT = 64;
  constexpr int KLD = DK + 8, VLD = DV + 8;
  __shared__ __align__(16) uint16_t ks[KT * KLD];
  __shared__ __align__(16) uint16_t vs[KT * VLD];
  typedef uint32_t vfrag __attribute__((ext_vector_type(NV / 2)));
  const int tid = threadIdx.x, lane = tid & 63, l32 = lane & 31, lh = lane >> 5;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int tile = (int)gridDim.x - 1 - (int)blockIdx.x;      // the longest key ranges first
  const int g = blockIdx.y;
  const int64_t b = blockIdx.z;
  const int col0 = *a.col_ptr, start = a.starts[b];
  const unsigned rows = (unsigned)(a.T * a.R);
  const unsigned row0 = (unsigned)tile * 128 + wave * 32, qrow = row0 + l32;
  const bool qvalid = qrow < rows;
  const unsigned qc = min(qrow, rows - 1);
  const int tq = (int)(qc / a.R), rq = (int)(qc % a.R), head = g * a.R + rq;
  const int c_n = col0 + tq;                                   // (the host checks col + T <= S where it can)
  const int w_lo = col0 + (int)(min(row0, rows - 1) / a.R), w_hi = col0 + (int)(min(row0 + 31, rows - 1) / a.R);
  const int t_hi = min(col0 + (int)(min((unsigned)tile * 128 + 127, rows - 1) / a.R), (int)a.S - 1);
  const uint16_t* q = reinterpret_cast<const uint16_t*>(a.q) + ((b * a.T + tq) * a.H + head) * DK;
  u32x4 qf[KD];
#pragma unroll
  for (int j = 0; j < KD; ++j) qf[j] = *reinterpret_cast<const u32x4*>(q + j * 16 + lh * 8);
  f32x16 O[NV];
#pragma unroll
  for (int j = 0; j < NV; ++j)
#pragma unroll
    for (int i = 0; i < 16; ++i) O[j][i] = 0.f;
  float m_run = kNegBig, l_run = 0.f;
  const float sc2 = a.scale * kLog2e, factor = !BIAS && sc2 > 0.f ? sc2 : 1.0f;
  // columns that this position, and the first and last one of the wave, see first
  const int seen = BIAS ? first_seen(c_n, start, a.chunk) : start;
  const int w_first = BIAS ? first_seen(w_lo, start, a.chunk) : start, w_last = BIAS ? first_seen(w_hi, start, a.chunk) : start;
  const float slope2 = BIAS && a.slopes ? a.slopes[head] * kLog2e : 0.f;
  const rsrc_t rk = make_rsrc(reinterpret_cast<const uint16_t*>(a.k) + (b * a.G + g) * a.S * DK, (uint64_t)a.S * DK * 2);
  const rsrc_t rv = make_rsrc(reinterpret_cast<const uint16_t*>(a.v) + (b * a.G + g) * a.S * DV, (uint64_t)a.S * DV * 2);
  constexpr int KC = KT * DK / 8 / 256, VC = KT * DV / 8 / 256;   // 16-byte chunks per thread
  u32x4 kr[KC], vr[VC];
  auto fetch = [&](int kb) {
#pragma unroll
    for (int c = 0; c < KC; ++c) {
      const int i = c * 256 + tid, r = i / (DK / 8), ch = i % (DK / 8);
      kr[c] = __builtin_amdgcn_raw_buffer_load_b128(rk, (uint32_t)((kb + r) * DK + ch * 8) * 2u, 0, 0);
    }
#pragma unroll
    for (int c = 0; c < VC; ++c) {
      const int i = c * 256 + tid, r = i / (DV / 8), ch = i % (DV / 8);
      vr[c] = __builtin_amdgcn_raw_buffer_load_b128(rv, (uint32_t)((kb + r) * DV + ch * 8) * 2u, 0, 0);
    }
  };
  int kb0 = max(start, 0) & ~(KT - 1);
  if constexpr (BIAS) kb0 = first_seen(col0 + (int)(min((unsigned)tile * 128, rows - 1) / a.R), start, a.chunk) & ~(KT - 1);
  if (kb0 <= t_hi) fetch(kb0);
  for (int kb = kb0; kb <= t_hi; kb += KT) {
    __syncthreads();
#pragma unroll
    for (int c = 0; c < KC; ++c) {
      const int i = c * 256 + tid;
      *reinterpret_cast<u32x4*>(&ks[(i / (DK / 8)) * KLD + (i % (DK / 8)) * 8]) = kr[c];
    }
#pragma unroll
    for (int c = 0; c < VC; ++c) {
      const int i = c * 256 + tid;
      *reinterpret_cast<u32x4*>(&vs[(i / (DV / 8)) * VLD + (i % (DV / 8)) * 8]) = vr[c];
    }
    __syncthreads();
    if (kb + KT <= t_hi) fetch(kb + KT);
    if (kb > w_hi || (BIAS && kb + KT - 1 < w_first)) continue;   // (wave-uniform: nothing visible in this tile)
    f32x16 st[2];
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
#pragma unroll
      for (int i = 0; i < 16; ++i) st[hf][i] = 0.f;
#pragma unroll
      for (int j = 0; j < KD; ++j)
        st[hf] = mfma32(*reinterpret_cast<const u32x4*>(&ks[(hf * 32 + l32) * KLD + j * 16 + lh * 8]), qf[j], st[hf]);
    }
    if constexpr (BIAS) {
      const float far = slope2 * (float)(kb + 4 * lh - c_n);
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int i = 0; i < 16; ++i) st[hf][i] = __builtin_fmaf(st[hf][i], sc2, __builtin_fmaf(slope2, (float)(hf * 32 + 8 * (i >> 2) + (i & 3)), far));
    } else if (sc2 <= 0.f) {   // (uniform; the maximum below is taken over unscaled scores)
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int i = 0; i < 16; ++i) st[hf][i] *= sc2;
    }
    // register 4 b + e of st[hf]: key kb + 32 hf + 8 b + 4 lh + e
    if (!(kb >= w_last && kb + KT - 1 <= w_lo)) {
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          const int key = kb + hf * 32 + 8 * (i >> 2) + 4 * lh + (i & 3);
          if (key < seen || key > c_n) st[hf][i] = -__builtin_inff();
        }
    }
    float mx = st[0][0];
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int i = 0; i < 16; ++i) mx = fmaxf(mx, st[hf][i]);
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float m_new = fmaxf(m_run, mx * factor);
    const float alpha = exp2_hw(m_run - m_new);
    m_run = m_new;
    float psum = 0.f;
    u32x4 pf[2][2];
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
      float p[16];
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        p[i] = exp2_hw(__builtin_fmaf(st[hf][i], factor, -m_new));   // (exp2(-inf) = 0: a masked key)
        psum += p[i];
      }
#pragma unroll
      for (int s = 0; s < 2; ++s)
        pf[hf][s] = u32x4{pack2bf(p[8 * s], p[8 * s + 1]), pack2bf(p[8 * s + 2], p[8 * s + 3]), pack2bf(p[8 * s + 4], p[8 * s + 5]),
                          pack2bf(p[8 * s + 6], p[8 * s + 7])};
    }
    l_run = l_run * alpha + psum;
    if (__builtin_amdgcn_ballot_w64(alpha != 1.0f) != 0) {
#pragma unroll
      for (int j = 0; j < NV; ++j)
#pragma unroll
        for (int i = 0; i < 16; ++i) O[j][i] *= alpha;
    }
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        // k index 8 lh + 4 b + e of this step <-> key 16 s + 8 b + 4 lh + e; lane l32 holds value
        // columns NV l32 + j of its eight keys
        vfrag v[8];
#pragma unroll
        for (int i = 0; i < 8; ++i)
          v[i] = *reinterpret_cast<const vfrag*>(&vs[(hf * 32 + 16 * s + 8 * (i >> 2) + 4 * lh + (i & 3)) * VLD + NV * l32]);
#pragma unroll
        for (int j = 0; j < NV; ++j) {
          const uint32_t sel = (j & 1) ? 0x07060302u : 0x05040100u;
          u32x4 af;
#pragma unroll
          for (int r = 0; r < 4; ++r) af[r] = __builtin_amdgcn_perm(v[2 * r + 1][j >> 1], v[2 * r][j >> 1], sel);
          O[j] = mfma32(af, pf[hf][s], O[j]);
        }
      }
  }
  if (!qvalid) return;
  l_run += __shfl_xor(l_run, 32, 64);
  const float w = finish_scale(m_run, l_run, a.sinks != nullptr, a.sinks ? a.sinks[head] : 0.f);
  // register 4 b + e of O[j]: value column NV (8 b + 4 lh + e) + j: runs of 4 NV columns
  uint16_t* out = reinterpret_cast<uint16_t*>(a.out);
  const int64_t orow = b * a.T + tq, cb = (int64_t)head * a.out_head;
  const bool vec = a.dv % 8 == 0 && a.out_head % 8 == 0 && a.out_ld % 8 == 0;
#pragma unroll
  for (int bb = 0; bb < 4; ++bb) {
    const int d0 = NV * (8 * bb + 4 * lh);
    float x[4 * NV];
#pragma unroll
    for (int e = 0; e < 4; ++e)
#pragma unroll
      for (int j = 0; j < NV; ++j) x[e * NV + j] = O[j][4 * bb + e] * w;
#pragma unroll
    for (int c = 0; c < 4 * NV; c += 8) {
      if (d0 + c >= a.dv) continue;
      const int64_t col = cb + d0 + c;
      if (vec) {
        *reinterpret_cast<u32x4*>(out + (a.out_frag ? frag_index(orow, col, a.out_ld) : orow * a.out_ld + col)) =
            u32x4{pack2bf(x[c], x[c + 1]), pack2bf(x[c + 2], x[c + 3]), pack2bf(x[c + 4], x[c + 5]), pack2bf(x[c + 6], x[c + 7])};
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e)
          if (d0 + c + e < a.dv)
            out[a.out_frag ? frag_index(orow, col + e, a.out_ld) : orow * a.out_ld + col + e] = f2bf(x[c + e]);
      }
    }
  }
}

template <int KS, int NH, int NJ>
void launch_step(hipStream_t st, const SinkArgs& a) {
  const unsigned qts = (unsigned)cdiv(a.T * a.R, 16);
  const dim3 grid((unsigned)a.n_chunks, (unsigned)a.G * qts, (unsigned)a.B);
  if (a.slopes || a.chunk > 0) hipLaunchKernelGGL((sink_attn_step_kernel<KS, NH, NJ, true>), grid, dim3(64), 0, st, a);
  else hipLaunchKernelGGL((sink_attn_step_kernel<KS, NH, NJ, false>), grid, dim3(64), 0, st, a);
}
template <int KS>
int launch_step_v(hipStream_t st, const SinkArgs& a) {
  if (a.dvp == 64) launch_step<KS, 1, 4>(st, a);
  else if (a.dvp == 128) launch_step<KS, 1, 8>(st, a);
  else launch_step<KS, 2, 8>(st, a);
  TNX_CHECK_LAUNCH("sink_attn_step");
  return TNX_OK;
}
template <int KD, int NV>
void launch_tile(hipStream_t st, const SinkArgs& a) {
  const dim3 grid((unsigned)cdiv(a.T * a.R, 128), (unsigned)a.G, (unsigned)a.B);
  if (a.slopes || a.chunk > 0) hipLaunchKernelGGL((sink_attn_tile_kernel<KD, NV, true>), grid, dim3(256), 0, st, a);
  else hipLaunchKernelGGL((sink_attn_tile_kernel<KD, NV, false>), grid, dim3(256), 0, st, a);
}
template <int KD>
int launch_tile_v(hipStream_t st, const SinkArgs& a) {
  if (a.dvp == 64) launch_tile<KD, 2>(st, a);
  else if (a.dvp == 128) launch_tile<KD, 4>(st, a);
  else launch_tile<KD, 8>(st, a);
  TNX_CHECK_LAUNCH("sink_attn_tile");
  return TNX_OK;
}
bool mfma_sizes(int dkp, int dvp) {
  return (dkp == 64 || dkp == 128 || dkp == 192 || dkp == 256) && (dvp == 64 || dvp == 128 || dvp == 256);
}

}  // namespace

extern "C" int tnx_sink_attn_pad(int dim, int is_value) {
  if (dim <= 0) return 0;
  if (is_value) return dim <= 64 ? 64 : dim <= 128 ? 128 : dim <= 256 ? 256 : dim;
  return dim <= 256 ? (dim + 63) / 64 * 64 : dim;
}

extern "C" size_t tnx_sink_attn_ws_bytes(int64_t B, int64_t T, int64_t S, int H, int dvp, int kv_chunk) {
  if (kv_chunk <= 0 || kv_chunk >= S) return 0;
  return (size_t)(B * T * H) * (size_t)cdiv(S, kv_chunk) * (size_t)(dvp + 2) * sizeof(float);
}

extern "C" int tnx_sink_attn(void* stream, const tnx_sink_attn_desc* d) {
  TNX_REQUIRE(d, "sink_attn: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->T > 0 && d->S >= d->T && d->H > 0 && d->G > 0 && d->H % d->G == 0, "sink_attn: bad shape");
  TNX_REQUIRE(d->dk > 0 && d->dv > 0 && d->dkp >= d->dk && d->dvp >= d->dv && d->dv <= 2048, "sink_attn: bad head sizes");
  TNX_REQUIRE(d->q && d->kcache && d->vcache && d->starts && d->col_ptr && d->out, "sink_attn: null pointer");
  TNX_REQUIRE(d->out_head == 0 || d->out_head >= d->dv, "sink_attn: short output heads");
  TNX_REQUIRE(d->out_ld >= (int64_t)d->H * (d->out_head ? d->out_head : d->dv), "sink_attn: short output rows");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "sink_attn: bad dtype %d", d->dtype);
  TNX_REQUIRE(d->B <= 65535, "sink_attn: too many rows");
  SinkArgs a;
  a.B = d->B; a.T = d->T; a.S = d->S; a.H = d->H; a.G = d->G; a.R = d->H / d->G; a.dk = d->dk; a.dv = d->dv; a.dkp = d->dkp;
  a.dvp = d->dvp; a.scale = d->scale; a.q = d->q; a.k = d->kcache; a.v = d->vcache; a.sinks = d->sinks; a.starts = d->starts;
  a.col_ptr = d->col_ptr; a.ws = d->ws; a.out = d->out; a.out_ld = d->out_ld; a.out_frag = d->out_frag;
  a.out_head = d->out_head ? d->out_head : d->dv;
  a.slopes = d->slopes; a.chunk = d->chunk > 0 && d->chunk < d->S ? d->chunk : 0;
  // one position sees at most its chunk; the splits begin at a block's edge in front of it
  const int64_t span = a.chunk > 0 && d->T == 1 && a.chunk + 31 < d->S ? a.chunk + 31 : d->S;
  a.kv_chunk = d->kv_chunk; a.n_chunks = d->kv_chunk > 0 && d->kv_chunk < span ? (int)cdiv(span, d->kv_chunk) : 1;
  hipStream_t st = as_stream(stream);
  const bool mfma = d->dtype == TNX_BF16 && mfma_sizes(d->dkp, d->dvp) && (uint64_t)d->S * (uint64_t)(d->dkp > d->dvp ? d->dkp : d->dvp) * 2 < (1ull << 31);
  if (!mfma) {
    // one work-group per (query position, head)
    TNX_REQUIRE(d->B * d->T <= 65535, "sink_attn: at most 65535 query rows per call at these sizes");
    const dim3 grid((unsigned)d->H, (unsigned)(d->B * d->T));
    if (d->dtype == TNX_BF16) hipLaunchKernelGGL(sink_attn_any_kernel<uint16_t>, grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL(sink_attn_any_kernel<float>, grid, dim3(256), 0, st, a);
    TNX_CHECK_LAUNCH("sink_attn_any");
    return TNX_OK;
  }
  if (d->T * a.R <= 64 || a.n_chunks > 1) {
    TNX_REQUIRE(a.n_chunks == 1 || a.ws, "sink_attn: a split key range needs a workspace");
    TNX_REQUIRE(a.n_chunks == 1 || a.kv_chunk % 32 == 0, "sink_attn: kv_chunk must be a multiple of 32");
    TNX_REQUIRE((int64_t)a.G * cdiv(d->T * a.R, 16) <= 65535, "sink_attn: too many query tiles");
    int rc;
    switch (d->dkp) {
      case 64: rc = launch_step_v<2>(st, a); break;
      case 128: rc = launch_step_v<4>(st, a); break;
      case 192: rc = launch_step_v<6>(st, a); break;
      default: rc = launch_step_v<8>(st, a); break;
    }
    if (rc || a.n_chunks == 1) return rc;
    hipLaunchKernelGGL(sink_attn_merge_kernel, dim3((unsigned)(d->B * d->T * d->H)), dim3(128), (size_t)a.n_chunks * 4, st, a);
    TNX_CHECK_LAUNCH("sink_attn_merge");
    return TNX_OK;
  }
  switch (d->dkp) {
    case 64: return launch_tile_v<4>(st, a);
    case 128: return launch_tile_v<8>(st, a);
    case 192: return launch_tile_v<12>(st, a);
    default: return launch_tile_v<16>(st, a);
  }
}
