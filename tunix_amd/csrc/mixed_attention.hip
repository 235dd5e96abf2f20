// Causal grouped-query attention whose softmax weights are mixed between the heads before they meet the values:
//   out_h = (sum_g talk[h, g] softmax(scale q_g k)) V_h  [* sigmoid(gate_h)],
// V_h the values of head h's own kv head.  Caches K [B, G, S, dkp] and V [B, G, S, dvp] have zero-padded rows; a row's
// keys start at starts[b].  The mixing needs finished weights of every head, so the softmax denominators come first.
// Scores, softmax and mixed weights are fp32; softmax weights enter the mixing product as a high and a low bf16 part, and
// mixed weights the product with the values as bf16.
//
//   mixed_stats_kernel    many positions: logarithm of every (position, head)'s denominator
//   mixed_tile_kernel     many positions: 16 positions x all heads per work-group; weights and mixed weights pass through
//                         LDS, each wave computes the scores and the output of its own heads
//   mixed_score_kernel    one position per sequence: scores and denominators of key chunks, keys read once
//   mixed_value_kernel    one position per sequence: weights, mixing and values of a key chunk, values read once
//   mixed_join_kernel     sum over the chunks, gate
//   mixed_any_kernel      any sizes and fp32: plain loops
#include <string.h>

#include <mutex>

#include "decoder.h"

namespace {

struct MixedArgs {
  int64_t B, T, S;
  int H, G, R, dk, dv, dkp, dvp;
  float scale;
  const void* q;
  const void* k;
  const void* v;
  const float* talk;       // [H, H]
  const int32_t* starts;   // [B]
  const int32_t* col_ptr;
  int kv_chunk, n_chunks;  // one position: keys of a work-group of mixed_value_kernel
  int s_chunk, s_chunks;   // the same of mixed_score_kernel
  float* lse;              // many positions: [B * T, H], log2 of the denominators
  float* scores;           // one position: [B, H, Sp], log2 units
  float* ml;               // [B, H, s_chunks, 2]: maximum and sum of a chunk
  float* part;             // [B, n_chunks, H, dvp]
  int64_t Sp;
  int gated;
  int64_t g_off;
  void* out;
  int64_t out_ld;
  int out_frag;
};

constexpr float kNegBig = -1.0e30f;
constexpr float kLog2e = 1.4426950408889634f;
__device__ __forceinline__ float exp2_hw(float x) { return __builtin_amdgcn_exp2f(x); }

// ---- any sizes ----------------------------------------------------------------------------------
// One work-group per position: denominators head by head, then 64 keys at a time the weights of all heads, their mixture
// and its product with the values, all in LDS.
template <typename T>
__global__ __launch_bounds__(256) void mixed_any_kernel(const MixedArgs a, const RowSrc<T> gate) {
  extern __shared__ float sm[];
  float* p = sm;                         // [H][64]
  float* w = p + a.H * 64;               // [H][64]
  float* top = w + a.H * 64;             // [H]
  float* den = top + a.H;                // [H]
  float* o = den + a.H;                  // [H * dv]
  const int64_t row = blockIdx.x, b = row / a.T, t = row % a.T;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int last = min(*a.col_ptr + (int)t, (int)a.S - 1), first = a.starts[b];
  const T* q = reinterpret_cast<const T*>(a.q) + row * a.H * a.dkp;
  const T* k = reinterpret_cast<const T*>(a.k) + b * a.G * a.S * a.dkp;
  const T* v = reinterpret_cast<const T*>(a.v) + b * a.G * a.S * a.dvp;
  auto score = [&](int h, int key) {
    const T* kr = k + ((int64_t)(h / a.R) * a.S + key) * a.dkp;
    float d = 0.f;
    for (int i = 0; i < a.dk; ++i) d += ld_elem(q, (int64_t)h * a.dkp + i) * ld_elem(kr, i);
    return d * a.scale;
  };
  for (int h = wave; h < a.H; h += 4) {
    float m = kNegBig, l = 0.f;
    for (int key = first + lane; key <= last; key += 64) {
      const float s = score(h, key), mn = fmaxf(m, s);
      l = l * expf(m - mn) + expf(s - mn);
      m = mn;
    }
    const float mt = wave_max(m);
    l = wave_sum(l * expf(m - mt));
    if (lane == 0) {
      top[h] = mt;
      den[h] = l;
    }
  }
  for (int i = tid; i < a.H * a.dv; i += 256) o[i] = 0.f;
  for (int k0 = first; k0 <= last; k0 += 64) {
    const int n = min(64, last - k0 + 1);
    __syncthreads();
    for (int h = wave; h < a.H; h += 4) p[h * 64 + lane] = lane < n ? expf(score(h, k0 + lane) - top[h]) / den[h] : 0.f;
    __syncthreads();
    for (int i = tid; i < a.H * 64; i += 256) {
      float s = 0.f;
      for (int g = 0; g < a.H; ++g) s += a.talk[(i >> 6) * a.H + g] * p[g * 64 + (i & 63)];
      w[i] = s;
    }
    __syncthreads();
    for (int i = tid; i < a.H * a.dv; i += 256) {
      const int h = i / a.dv;
      const T* vr = v + ((int64_t)(h / a.R) * a.S + k0) * a.dvp + i % a.dv;
      float s = o[i];
      for (int j = 0; j < n; ++j) s += w[h * 64 + j] * ld_elem(vr, (int64_t)j * a.dvp);
      o[i] = s;
    }
  }
  T* out = reinterpret_cast<T*>(a.out);
  for (int i = tid; i < a.H * a.dv; i += 256)   // (a thread reads what it wrote)
    st_elem(out, a.out_frag ? frag_index(row, i, a.out_ld) : row * a.out_ld + i, a.gated ? o[i] * sigmoid_f32(gate.get(row, a.g_off + i)) : o[i]);
}

// ---- many positions: denominators -----------------------------------------------------------------
// 128 query rows = (position, head of the group) pairs per work-group, keys of 64 slots staged in LDS; S^T = K . Q^T, so
// that a lane owns one query.
template <int KD>   // 16-deep k-steps of the head size
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2, 4))) void mixed_stats_kernel(const MixedArgs a) {
  constexpr int DK = KD * 16, KT = 64, KLD = DK + 8;
  __shared__ __align__(16) uint16_t ks[KT * KLD];
  const int tid = threadIdx.x, lane = tid & 63, l32 = lane & 31, lh = lane >> 5;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int tile = (int)gridDim.x - 1 - (int)blockIdx.x;      // the longest key ranges first
  const int g = blockIdx.y;
  const int64_t b = blockIdx.z;
  const int col0 = *a.col_ptr, start = a.starts[b];
  const unsigned rows = (unsigned)(a.T * a.R);
  const unsigned row0 = (unsigned)tile * 128 + wave * 32, qrow = row0 + l32;
  const unsigned qc = min(qrow, rows - 1);
  const int tq = (int)(qc / a.R), head = g * a.R + (int)(qc % a.R);
  const int c_n = col0 + tq;
  const int w_lo = col0 + (int)(min(row0, rows - 1) / a.R), w_hi = col0 + (int)(min(row0 + 31, rows - 1) / a.R);
  const int t_hi = min(col0 + (int)(min((unsigned)tile * 128 + 127, rows - 1) / a.R), (int)a.S - 1);
  const uint16_t* q = reinterpret_cast<const uint16_t*>(a.q) + ((b * a.T + tq) * a.H + head) * DK;
  u32x4 qf[KD];
#pragma unroll
  for (int j = 0; j < KD; ++j) qf[j] = *reinterpret_cast<const u32x4*>(q + j * 16 + lh * 8);
  float m_run = kNegBig, l_run = 0.f;
  const float sc2 = a.scale * kLog2e;
  const rsrc_t rk = make_rsrc(reinterpret_cast<const uint16_t*>(a.k) + (b * a.G + g) * a.S * DK, (uint64_t)a.S * DK * 2);
  constexpr int KC = KT * DK / 8 / 256;   // 16-byte chunks per thread
  u32x4 kr[KC];
  auto fetch = [&](int kb) {
#pragma unroll
    for (int c = 0; c < KC; ++c) {
      const int i = c * 256 + tid, r = i / (DK / 8), ch = i % (DK / 8);
      kr[c] = __builtin_amdgcn_raw_buffer_load_b128(rk, (uint32_t)((kb + r) * DK + ch * 8) * 2u, 0, 0);
    }
  };
  const int kb0 = max(start, 0) & ~(KT - 1);
  if (kb0 <= t_hi) fetch(kb0);
  for (int kb = kb0; kb <= t_hi; kb += KT) {
    __syncthreads();
#pragma unroll
    for (int c = 0; c < KC; ++c) {
      const int i = c * 256 + tid;
      *reinterpret_cast<u32x4*>(&ks[(i / (DK / 8)) * KLD + (i % (DK / 8)) * 8]) = kr[c];
    }
    __syncthreads();
    if (kb + KT <= t_hi) fetch(kb + KT);
    if (kb > w_hi) continue;                                   // (wave-uniform: nothing visible in this tile)
    f32x16 st[2];
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
#pragma unroll
      for (int i = 0; i < 16; ++i) st[hf][i] = 0.f;
#pragma unroll
      for (int j = 0; j < KD; ++j)
        st[hf] = mfma32(*reinterpret_cast<const u32x4*>(&ks[(hf * 32 + l32) * KLD + j * 16 + lh * 8]), qf[j], st[hf]);
#pragma unroll
      for (int i = 0; i < 16; ++i) st[hf][i] *= sc2;
    }
    // register 4 b + e of st[hf]: key kb + 32 hf + 8 b + 4 lh + e
    if (!(kb >= start && kb + KT - 1 <= w_lo)) {
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          const int key = kb + hf * 32 + 8 * (i >> 2) + 4 * lh + (i & 3);
          if (key < start || key > c_n) st[hf][i] = -__builtin_inff();
        }
    }
    float mx = st[0][0];
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int i = 0; i < 16; ++i) mx = fmaxf(mx, st[hf][i]);
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float m_new = fmaxf(m_run, mx), alpha = exp2_hw(m_run - m_new);
    m_run = m_new;
    float psum = 0.f;
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int i = 0; i < 16; ++i) psum += exp2_hw(st[hf][i] - m_new);   // (exp2(-inf) = 0: a masked key)
    l_run = l_run * alpha + psum;
  }
  l_run += __shfl_xor(l_run, 32, 64);
  if (qrow < rows && lh == 0) a.lse[(b * a.T + tq) * a.H + head] = l_run > 0.f ? m_run + __log2f(l_run) : -kNegBig;
}

// 16 positions of one head, [16][DV] in LDS, gated and rounded
template <int DV>
__device__ __forceinline__ void store_head(const MixedArgs& a, const RowSrc<uint16_t>& gate, const float* ob, uint16_t* out, int64_t b, int t0, int head, int lane,
                                           bool vec) {
#pragma unroll 1
  for (int it = lane; it < 16 * (DV / 8); it += 64) {
    const int t = t0 + it / (DV / 8), d = it % (DV / 8) * 8;
    if (t >= a.T || d >= a.dv) continue;
    const int64_t row = b * a.T + t, col = (int64_t)head * a.dv + d;
    const f32x4 u = *reinterpret_cast<const f32x4*>(ob + it * 8), v = *reinterpret_cast<const f32x4*>(ob + it * 8 + 4);
    float f[8] = {u[0], u[1], u[2], u[3], v[0], v[1], v[2], v[3]};
    if (vec) {
      if (a.gated) {
        float z[8];
        get8(gate, row, a.g_off + col, z);
#pragma unroll
        for (int j = 0; j < 8; ++j) f[j] *= sigmoid_f32(z[j]);
      }
      put8(out + (a.out_frag ? frag_index(row, col, a.out_ld) : row * a.out_ld + col), f);
      continue;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (d + j < a.dv)
        out[a.out_frag ? frag_index(row, col + j, a.out_ld) : row * a.out_ld + col + j] = f2bf(f[j] * (a.gated ? sigmoid_f32(gate.get(row, a.g_off + col + j)) : 1.f));
  }
}

// ---- many positions: weights, mixing, values ---------------------------------------------------------
// A work-group of NW waves takes 16 positions of one sequence and all heads, 32 keys at a time.  Wave w owns heads w HW ..:
//   1. S^T = K . Q^T of its heads (16x16x32 MFMAs: a lane has one position and eight keys), weights to LDS as
//      [key][position][head], high and low parts;
//   2. mixing: of 32 / NW keys for all heads, talk (A operand) times weights (B operand, the head as k), to LDS as
//      [head][position][key];
//   3. O = W . V of its heads; value rows as in mixed_value_kernel.
// Two barriers a turn: the weights of a turn are read before its second one, the mixed weights before the next turn's first.
// ONE: the heads of a wave share their kv head, so that its keys and values are requested a phase ahead.
template <int KS, int NH, int NJ, int HW, int NW, bool ONE>   // 32-deep k-steps; halves and value columns per lane and half; heads of a wave
__global__ __launch_bounds__(64 * NW) __attribute__((amdgpu_waves_per_eu(1, 2))) void mixed_tile_kernel(const MixedArgs a, const RowSrc<uint16_t> gate) {
  constexpr int DK = KS * 32, DV = NH * NJ * 16, HS = NW * HW;
  constexpr int HT = (HS + 15) / 16, GP = HT * 16;                 // 16-row tiles of heads; head slots
  constexpr int PLD = GP + 8, KSTR = 16 * PLD + 8, WLD = 40, KPW = 32 / NW;
  typedef uint32_t vfrag __attribute__((ext_vector_type(NJ / 2)));
  extern __shared__ __align__(16) uint16_t lds[];
  uint16_t* ph = lds;                        // [32][KSTR]
  uint16_t* pl = ph + 32 * KSTR;
  uint16_t* ws = pl + 32 * KSTR;             // [GP][16][WLD]
  const int tid = threadIdx.x, lane = tid & 63, lm = lane & 15, lq = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  // sequences fastest: with a multiple of eight of them, the work-groups of one share an XCD and its keys stay in that L2
  const int tile = (int)gridDim.y - 1 - (int)blockIdx.y;           // the longest key ranges first
  const int64_t b = blockIdx.x;
  const int col0 = *a.col_ptr, start = a.starts[b];
  const int tp = tile * 16 + lm, tq = min(tp, (int)a.T - 1);       // this lane's position as a column
  const int c_n = col0 + tq, w_lo = col0 + tile * 16, t_hi = min(col0 + min(tile * 16 + 15, (int)a.T - 1), (int)a.S - 1);
  for (int i = tid; i < 32 * KSTR; i += 64 * NW) reinterpret_cast<uint32_t*>(ph)[i] = 0u;   // (both parts; slots behind the last head stay zero)
  u32x4 qf[HW][KS], tf[HT];
  float lse[HW];
#pragma unroll
  for (int hh = 0; hh < HW; ++hh) {
    const int g = min(wave * HW + hh, a.H - 1);
    const uint16_t* q = reinterpret_cast<const uint16_t*>(a.q) + ((b * a.T + tq) * a.H + g) * DK;
#pragma unroll
    for (int j = 0; j < KS; ++j) qf[hh][j] = *reinterpret_cast<const u32x4*>(q + j * 32 + lq * 8);
    lse[hh] = a.lse[(b * a.T + tq) * a.H + g];
  }
#pragma unroll
  for (int ht = 0; ht < HT; ++ht) {
    float f[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int h = ht * 16 + lm, g = lq * 8 + e;
      f[e] = h < a.H && g < a.H ? a.talk[h * a.H + g] : 0.f;
    }
    tf[ht] = u32x4{pack2bf(f[0], f[1]), pack2bf(f[2], f[3]), pack2bf(f[4], f[5]), pack2bf(f[6], f[7])};
  }
  f32x4 O[HW][NH][NJ];
#pragma unroll
  for (int hh = 0; hh < HW; ++hh)
#pragma unroll
    for (int h = 0; h < NH; ++h)
#pragma unroll
      for (int j = 0; j < NJ; ++j) O[hh][h][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const float sc2 = a.scale * kLog2e;
  const rsrc_t rk = make_rsrc(reinterpret_cast<const uint16_t*>(a.k) + b * a.G * a.S * DK, (uint64_t)a.G * a.S * DK * 2);
  const rsrc_t rv = make_rsrc(reinterpret_cast<const uint16_t*>(a.v) + b * a.G * a.S * DV, (uint64_t)a.G * a.S * DV * 2);
  // (rows past a kv head's slots are the next head's, or zeros behind the last: their weights are zero)
  u32x4 kf[2][KS];
  auto load_k = [&](int c, int kb) {
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int j = 0; j < KS; ++j)
        kf[s][j] = __builtin_amdgcn_raw_buffer_load_b128(rk, (uint32_t)((c * (int)a.S + kb + s * 16 + lm) * DK + j * 32 + lq * 8) * 2u, 0, 0);
  };
  vfrag vf[NH][8];
  auto load_v = [&](int c, int kb) {
#pragma unroll
    for (int s = 0; s < 8; ++s)
#pragma unroll
      for (int h = 0; h < NH; ++h) {
        const uint32_t o = (uint32_t)((c * (int)a.S + kb + 8 * lq + s) * DV + h * 16 * NJ + NJ * lm) * 2u;
        if constexpr (NJ == 8) vf[h][s] = __builtin_amdgcn_raw_buffer_load_b128(rv, o, 0, 0);
        else vf[h][s] = __builtin_amdgcn_raw_buffer_load_b64(rv, o, 0, 0);
      }
  };
  const bool busy = wave * HW < a.H;                               // (wave-uniform)
  const int c_first = min(wave * HW, a.H - 1) / a.R;
  const int kb0 = max(start, 0) & ~31;
  if (busy && kb0 <= t_hi) load_k(c_first, kb0);
  __syncthreads();
  for (int kb = kb0; kb <= t_hi; kb += 32) {
    if (busy) {
      const bool whole = kb >= start && kb + 31 <= w_lo;           // (uniform) every key visible to every position
      float p[HW][8];
      int c = c_first;
#pragma unroll
      for (int hh = 0; hh < HW; ++hh) {
        const int g = wave * HW + hh;
        if (g >= a.H) {
#pragma unroll
          for (int i = 0; i < 8; ++i) p[hh][i] = 0.f;
          continue;
        }
        if constexpr (!ONE) {
          if (g / a.R != c) {
            c = g / a.R;
            load_k(c, kb);
          }
        }
#pragma unroll
        for (int s = 0; s < 2; ++s) {
          f32x4 st = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int j = 0; j < KS; ++j) st = mfma16(kf[s][j], qf[hh][j], st);
#pragma unroll
          for (int i = 0; i < 4; ++i) p[hh][4 * s + i] = exp2_hw(__builtin_fmaf(st[i], sc2, -lse[hh]));
        }
        if (!whole)
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            const int key = kb + (i >> 2) * 16 + 4 * lq + (i & 3);
            if (key < start || key > c_n) p[hh][i] = 0.f;
          }
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int at = ((i >> 2) * 16 + 4 * lq + (i & 3)) * KSTR + lm * PLD + wave * HW;
        if constexpr (HW == 1) {
          const uint16_t hi = f2bf(p[0][i]);
          ph[at] = hi;
          pl[at] = f2bf(p[0][i] - bf2f(hi));
        } else if constexpr (HW == 2) {
          uint32_t hi, lo;
          split2(p[0][i], p[1][i], hi, lo);
          *reinterpret_cast<uint32_t*>(ph + at) = hi;
          *reinterpret_cast<uint32_t*>(pl + at) = lo;
        } else {
          uint32_t h0, l0, h1, l1;
          split2(p[0][i], p[1][i], h0, l0);
          split2(p[HW - 2][i], p[HW - 1][i], h1, l1);
          *reinterpret_cast<u32x2*>(ph + at) = u32x2{h0, h1};
          *reinterpret_cast<u32x2*>(pl + at) = u32x2{l0, l1};
        }
      }
      load_v(c_first, kb);
    }
    __syncthreads();
    {
      f32x4 w[HT][KPW];
#pragma unroll
      for (int kk = 0; kk < KPW; ++kk) {
        const int at = (wave * KPW + kk) * KSTR + lm * PLD + lq * 8;
        u32x4 fh = u32x4{0, 0, 0, 0}, fl = fh;
        if (GP == 32 || lq < GP / 8) {
          fh = *reinterpret_cast<const u32x4*>(ph + at);
          fl = *reinterpret_cast<const u32x4*>(pl + at);
        }
#pragma unroll
        for (int ht = 0; ht < HT; ++ht) w[ht][kk] = mfma16(tf[ht], fl, mfma16(tf[ht], fh, f32x4{0.f, 0.f, 0.f, 0.f}));
      }
#pragma unroll
      for (int ht = 0; ht < HT; ++ht)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          uint16_t* dst = ws + ((ht * 16 + 4 * lq + i) * 16 + lm) * WLD + wave * KPW;
          if constexpr (KPW == 8)
            *reinterpret_cast<u32x4*>(dst) = u32x4{pack2bf(w[ht][0][i], w[ht][1][i]), pack2bf(w[ht][2][i], w[ht][3][i]), pack2bf(w[ht][KPW - 4][i], w[ht][KPW - 3][i]),
                                                   pack2bf(w[ht][KPW - 2][i], w[ht][KPW - 1][i])};
          else
            *reinterpret_cast<u32x2*>(dst) = u32x2{pack2bf(w[ht][0][i], w[ht][1][i]), pack2bf(w[ht][2][i], w[ht][3][i])};
        }
    }
    __syncthreads();
    if (!busy) continue;
    load_k(c_first, min(kb + 32, t_hi & ~31));
    int c = c_first;
#pragma unroll
    for (int hh = 0; hh < HW; ++hh) {
      const int g = wave * HW + hh;
      if (g >= a.H) continue;
      if constexpr (!ONE) {
        if (g / a.R != c) {
          c = g / a.R;
          load_v(c, kb);
        }
      }
      const u32x4 wf = *reinterpret_cast<const u32x4*>(ws + (g * 16 + lm) * WLD + lq * 8);
#pragma unroll
      for (int h = 0; h < NH; ++h)
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
          const uint32_t sel = (j & 1) ? 0x07060302u : 0x05040100u;
          u32x4 bf;
#pragma unroll
          for (int r = 0; r < 4; ++r) bf[r] = __builtin_amdgcn_perm(vf[h][2 * r + 1][j >> 1], vf[h][2 * r][j >> 1], sel);
          O[hh][h][j] = mfma16(wf, bf, O[hh][h][j]);
        }
    }
  }
  // the heads' outputs through LDS, one head of a wave at a time, so that rows leave in runs of eight
  __syncthreads();
  if (!busy) return;
  float* ob = reinterpret_cast<float*>(lds) + wave * 16 * DV;
  uint16_t* out = reinterpret_cast<uint16_t*>(a.out);
  const bool vec = a.dv % 8 == 0 && a.out_ld % 8 == 0 && (!a.gated || (a.g_off % 8 == 0 && gate.ld % 8 == 0 && (gate.split <= 1 || gate.plane % 8 == 0)));
#pragma unroll
  for (int hh = 0; hh < HW; ++hh) {
    const int g = wave * HW + hh;
    if (g >= a.H) continue;
    // lane: positions 4 lq + i, value columns h * 16 NJ + NJ lm + j
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int h = 0; h < NH; ++h)
#pragma unroll
        for (int j = 0; j < NJ; j += 4)
          *reinterpret_cast<f32x4*>(ob + (4 * lq + i) * DV + h * 16 * NJ + NJ * lm + j) =
              f32x4{O[hh][h][j][i], O[hh][h][j + 1][i], O[hh][h][j + 2][i], O[hh][h][j + 3][i]};
    store_head<DV>(a, gate, ob, out, b, tile * 16, g, lane, vec);
  }
}

// ---- one position per sequence -------------------------------------------------------------------------
// One wave per (16 heads of a kv head, key chunk): S^T = K . q^T, 64 keys a turn, the next ones on their way.
template <int KS>
__global__ __launch_bounds__(64) __attribute__((amdgpu_waves_per_eu(1, KS > 4 ? 1 : 3))) void mixed_score_kernel(const MixedArgs a) {
  constexpr int DK = KS * 32;
  const int lane = threadIdx.x, lm = lane & 15, lq = lane >> 4;
  const int chunk = blockIdx.x, qts = (a.R + 15) / 16, g = blockIdx.y / qts, r = blockIdx.y % qts * 16 + lm;
  const int64_t b = blockIdx.z;
  const int start = a.starts[b], last = min(*a.col_ptr, (int)a.S - 1);
  const int k_lo = max(start, chunk * a.s_chunk), k_hi = min(last, chunk * a.s_chunk + a.s_chunk - 1);
  if (k_lo > k_hi) return;                                          // (its statistics are never read)
  const bool valid = r < a.R;
  const int head = g * a.R + min(r, a.R - 1);
  const uint16_t* q = reinterpret_cast<const uint16_t*>(a.q) + (b * a.H + head) * DK;
  u32x4 qf[KS];
#pragma unroll
  for (int j = 0; j < KS; ++j) qf[j] = *reinterpret_cast<const u32x4*>(q + j * 32 + lq * 8);
  const rsrc_t rk = make_rsrc(reinterpret_cast<const uint16_t*>(a.k) + (b * a.G + g) * a.S * DK, (uint64_t)a.S * DK * 2);
  struct Stage {
    u32x4 kf[4][KS];
  };
  auto load = [&](int kb, Stage& sg) {
#pragma unroll
    for (int s = 0; s < 4; ++s)
#pragma unroll
      for (int j = 0; j < KS; ++j)
        sg.kf[s][j] = __builtin_amdgcn_raw_buffer_load_b128(rk, (uint32_t)((kb + s * 16 + lm) * DK + j * 32 + lq * 8) * 2u, 0, kStreamOnce);
  };
  const float sc2 = a.scale * kLog2e;
  float m = kNegBig, l = 0.f;
  float* dst = a.scores + (b * a.H + head) * a.Sp;
  auto compute = [&](int kb, const Stage& sg) {
    f32x4 st[4];
    float mx = kNegBig;
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      st[s] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < KS; ++j) st[s] = mfma16(sg.kf[s][j], qf[j], st[s]);
      st[s] *= sc2;
      const int key = kb + s * 16 + 4 * lq;
      if (valid) *reinterpret_cast<f32x4*>(dst + key) = st[s];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if (key + i < k_lo || key + i > k_hi) st[s][i] = -__builtin_inff();
        mx = fmaxf(mx, st[s][i]);
      }
    }
    const float mn = fmaxf(m, mx);
    l *= exp2_hw(m - mn);
    m = mn;
#pragma unroll
    for (int s = 0; s < 4; ++s)
#pragma unroll
      for (int i = 0; i < 4; ++i) l += exp2_hw(st[s][i] - mn);
  };
  Stage sg[2];
  const int kb0 = k_lo & ~63, kb_last = k_hi & ~63;
  // (no load behind the last keys, and none under a condition inside the loop: its waits count exactly)
  load(kb0, sg[0]);
  int kb = kb0;
  for (; kb + 128 <= kb_last; kb += 128) {
    load(kb + 64, sg[1]);
    compute(kb, sg[0]);
    load(kb + 128, sg[0]);
    compute(kb + 64, sg[1]);
  }
  if (kb + 64 <= kb_last) {
    load(kb + 64, sg[1]);
    compute(kb, sg[0]);
    compute(kb + 64, sg[1]);
  } else {
    compute(kb, sg[0]);
  }
  // a head's four lanes
#pragma unroll
  for (int o = 16; o < 64; o <<= 1) {
    const float om = __shfl_xor(m, o, 64), ol = __shfl_xor(l, o, 64), mn = fmaxf(m, om);
    l = l * exp2_hw(m - mn) + ol * exp2_hw(om - mn);
    m = mn;
  }
  if (valid && lq == 0) {
    float* s = a.ml + ((b * a.H + head) * a.s_chunks + chunk) * 2;
    s[0] = m;
    s[1] = l;
  }
}

// One work-group per (sequence, key chunk): denominators from all chunks' statistics, weights and mixing of the chunk
// through LDS, then a wave per kv head streams the values; a lane holds value columns NJ lm .. of eight keys.
template <int NH, int NJ, int HT>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, 2))) void mixed_value_kernel(const MixedArgs a) {
  constexpr int DV = NH * NJ * 16, GP = HT * 16, PLD = GP + 8, KG = (GP + 31) / 32;
  typedef uint32_t vfrag __attribute__((ext_vector_type(NJ / 2)));
  extern __shared__ __align__(16) uint16_t lds[];
  __shared__ float lse[64];
  const int KC = a.kv_chunk, wld = KC + 8;
  uint16_t* ph = lds;                        // [KC][PLD]
  uint16_t* pl = ph + KC * PLD;
  uint16_t* ws = pl + KC * PLD;              // [GP][KC + 8]
  const int tid = threadIdx.x, lane = tid & 63, lm = lane & 15, lq = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int chunk = blockIdx.x;
  const int64_t b = blockIdx.y;
  const int start = a.starts[b], last = min(*a.col_ptr, (int)a.S - 1), base = chunk * KC;
  const int k_lo = max(start, base), k_hi = min(last, base + KC - 1);
  if (k_lo > k_hi) return;                                          // (its part is never read)
  // the first values are on their way while the weights are formed
  struct Stage {
    vfrag vf[NH][8];
  };
  const rsrc_t rv = make_rsrc(reinterpret_cast<const uint16_t*>(a.v) + b * a.G * a.S * DV, (uint64_t)a.G * a.S * DV * 2);
  auto load = [&](int c, int kb, Stage& s) {
#pragma unroll
    for (int k = 0; k < 8; ++k)
#pragma unroll
      for (int h = 0; h < NH; ++h) {
        const uint32_t o = (uint32_t)((c * (int)a.S + kb + 8 * lq + k) * DV + h * 16 * NJ + NJ * lm) * 2u;
        if constexpr (NJ == 8) s.vf[h][k] = __builtin_amdgcn_raw_buffer_load_b128(rv, o, 0, kStreamOnce);
        else s.vf[h][k] = __builtin_amdgcn_raw_buffer_load_b64(rv, o, 0, kStreamOnce);
      }
  };
  Stage sg[2];
  const int qts = (a.R + 15) / 16, kb0 = k_lo & ~31, kb_last = k_hi & ~31;
  if (wave < a.G * qts) load(wave / qts, kb0, sg[0]);
  {
    const int h = tid >> 2;
    float m = kNegBig, l = 0.f;
    if (h < a.H)
      for (int c = start / a.s_chunk + (tid & 3); c <= last / a.s_chunk; c += 4) {
        const float* s = a.ml + ((b * a.H + h) * a.s_chunks + c) * 2;
        const float mn = fmaxf(m, s[0]);
        l = l * exp2_hw(m - mn) + s[1] * exp2_hw(s[0] - mn);
        m = mn;
      }
#pragma unroll
    for (int o = 1; o < 4; o <<= 1) {
      const float om = __shfl_xor(m, o, 64), ol = __shfl_xor(l, o, 64), mn = fmaxf(m, om);
      l = l * exp2_hw(m - mn) + ol * exp2_hw(om - mn);
      m = mn;
    }
    if ((tid & 3) == 0) lse[h] = h < a.H ? m + __log2f(l) : -kNegBig;
  }
  __syncthreads();
  for (int it = tid; it < GP * (KC / 4); it += 256) {   // (heads fastest: they lie side by side in LDS)
    const int h = it % GP, k0 = it / GP * 4;
    f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
    if (h < a.H && base + k0 < a.Sp) s = *reinterpret_cast<const f32x4*>(a.scores + (b * a.H + h) * a.Sp + base + k0);
    const float e = lse[h];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int key = base + k0 + i;
      const float p = h < a.H && key >= k_lo && key <= k_hi ? exp2_hw(s[i] - e) : 0.f;
      const uint16_t hi = f2bf(p);
      ph[(k0 + i) * PLD + h] = hi;
      pl[(k0 + i) * PLD + h] = f2bf(p - bf2f(hi));
    }
  }
  __syncthreads();
#pragma unroll
  for (int ht = 0; ht < HT; ++ht) {
    u32x4 tf[KG];
#pragma unroll
    for (int kg = 0; kg < KG; ++kg) {
      float f[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int h = ht * 16 + lm, g = kg * 32 + lq * 8 + e;
        f[e] = h < a.H && g < a.H ? a.talk[h * a.H + g] : 0.f;
      }
      tf[kg] = u32x4{pack2bf(f[0], f[1]), pack2bf(f[2], f[3]), pack2bf(f[4], f[5]), pack2bf(f[6], f[7])};
    }
    for (int kt = wave; kt < KC / 16; kt += 4) {
      f32x4 w = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kg = 0; kg < KG; ++kg) {
        u32x4 fh = u32x4{0, 0, 0, 0}, fl = fh;
        if (kg * 32 + lq * 8 < GP) {
          fh = *reinterpret_cast<const u32x4*>(ph + (kt * 16 + lm) * PLD + kg * 32 + lq * 8);
          fl = *reinterpret_cast<const u32x4*>(pl + (kt * 16 + lm) * PLD + kg * 32 + lq * 8);
        }
        w = mfma16(tf[kg], fl, mfma16(tf[kg], fh, w));
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) ws[(ht * 16 + 4 * lq + i) * wld + kt * 16 + lm] = f2bf(w[i]);
    }
  }
  __syncthreads();
  for (int it = wave; it < a.G * qts; it += 4) {
    const int c = it / qts, r0 = it % qts * 16, head = c * a.R + min(r0 + lm, a.R - 1);
    if (it != wave) load(c, kb0, sg[0]);
    f32x4 O[NH][NJ];
#pragma unroll
    for (int h = 0; h < NH; ++h)
#pragma unroll
      for (int j = 0; j < NJ; ++j) O[h][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    auto compute = [&](int kb, const Stage& s) {
      const u32x4 wf = *reinterpret_cast<const u32x4*>(ws + head * wld + kb - base + lq * 8);
#pragma unroll
      for (int h = 0; h < NH; ++h)
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
          const uint32_t sel = (j & 1) ? 0x07060302u : 0x05040100u;
          u32x4 bf;
#pragma unroll
          for (int r = 0; r < 4; ++r) bf[r] = __builtin_amdgcn_perm(s.vf[h][2 * r + 1][j >> 1], s.vf[h][2 * r][j >> 1], sel);
          O[h][j] = mfma16(wf, bf, O[h][j]);
        }
    };
    int kb = kb0;
    for (; kb + 64 <= kb_last; kb += 64) {
      load(c, kb + 32, sg[1]);
      compute(kb, sg[0]);
      load(c, kb + 64, sg[0]);
      compute(kb + 32, sg[1]);
    }
    if (kb + 32 <= kb_last) {
      load(c, kb + 32, sg[1]);
      compute(kb, sg[0]);
      compute(kb + 32, sg[1]);
    } else {
      compute(kb, sg[0]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = r0 + 4 * lq + i;
      if (r >= a.R) continue;
      float* po = a.part + ((b * a.n_chunks + chunk) * a.H + c * a.R + r) * DV;
#pragma unroll
      for (int h = 0; h < NH; ++h)
#pragma unroll
        for (int j = 0; j < NJ; j += 4)
          *reinterpret_cast<f32x4*>(po + h * 16 * NJ + NJ * lm + j) = f32x4{O[h][j][i], O[h][j + 1][i], O[h][j + 2][i], O[h][j + 3][i]};
    }
  }
}

__global__ __launch_bounds__(256) void mixed_join_kernel(const MixedArgs a, const RowSrc<uint16_t> gate) {
  const int64_t b = blockIdx.x;
  const int start = a.starts[b], last = min(*a.col_ptr, (int)a.S - 1), c0 = start / a.kv_chunk, c1 = last / a.kv_chunk;
  uint16_t* out = reinterpret_cast<uint16_t*>(a.out);
  for (int i = blockIdx.y * 256 + threadIdx.x; i < a.H * a.dv; i += 256 * gridDim.y) {
    const int h = i / a.dv, d = i % a.dv;
    const float* p = a.part + (b * a.n_chunks * a.H + h) * a.dvp + d;
    float s = 0.f;
#pragma unroll 8
    for (int c = c0; c <= c1; ++c) s += p[(int64_t)c * a.H * a.dvp];
    if (a.gated) s *= sigmoid_f32(gate.get(b, a.g_off + i));
    out[a.out_frag ? frag_index(b, i, a.out_ld) : b * a.out_ld + i] = f2bf(s);
  }
}

constexpr int kMaxChunk = 320;
// ---- launches ---------------------------------------------------------------------------------------------
template <class K>
int raise_lds(K kern, size_t bytes) {
  const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
  if (e == hipSuccess) return TNX_OK;
  tnx_set_error("mixed_attn: cannot raise the dynamic LDS limit: %s", hipGetErrorString(e));
  return TNX_ELAUNCH;
}

template <int KS, int NH, int NJ, int HW, int NW, bool ONE>
int launch_tile_as(hipStream_t st, const MixedArgs& a, const RowSrc<uint16_t>& gate) {
  constexpr int GP = (NW * HW + 15) / 16 * 16;
  constexpr size_t kLoop = (size_t)(2 * 32 * (16 * (GP + 8) + 8) + GP * 16 * 40) * 2, kOut = (size_t)NW * 16 * NH * NJ * 16 * 4;
  constexpr size_t kLds = kLoop > kOut ? kLoop : kOut;
  static std::once_flag once;
  static int rc = TNX_OK;
  std::call_once(once, [] { rc = raise_lds(&mixed_tile_kernel<KS, NH, NJ, HW, NW, ONE>, kLds); });
  if (rc) return rc;
  hipLaunchKernelGGL((mixed_stats_kernel<2 * KS>), dim3((unsigned)cdiv(a.T * a.R, 128), (unsigned)a.G, (unsigned)a.B), dim3(256), 0, st, a);
  hipLaunchKernelGGL((mixed_tile_kernel<KS, NH, NJ, HW, NW, ONE>), dim3((unsigned)a.B, (unsigned)cdiv(a.T, 16)), dim3(64 * NW), kLds, st, a, gate);
  TNX_CHECK_LAUNCH("mixed_tile");
  return TNX_OK;
}
template <int KS, int NH, int NJ, int HW, int NW>
int launch_tile(hipStream_t st, const MixedArgs& a, const RowSrc<uint16_t>& gate) {
  if constexpr (HW > 1) {
    if (a.R % HW != 0) return launch_tile_as<KS, NH, NJ, HW, NW, false>(st, a, gate);
  }
  return launch_tile_as<KS, NH, NJ, HW, NW, true>(st, a, gate);
}
template <int KS, int NH, int NJ>
int launch_tile_heads(hipStream_t st, const MixedArgs& a, const RowSrc<uint16_t>& gate) {
  if (a.H <= 4) return launch_tile<KS, NH, NJ, 1, 4>(st, a, gate);
  if (a.H <= 8) return launch_tile<KS, NH, NJ, 2, 4>(st, a, gate);
  if constexpr (KS <= 4 && NH == 1) {
    if (a.H <= 16) return launch_tile<KS, NH, NJ, 4, 4>(st, a, gate);
    return launch_tile<KS, NH, NJ, 4, 8>(st, a, gate);
  } else {
    return launch_tile<KS, NH, NJ, 2, 8>(st, a, gate);
  }
}
template <int KS>
int launch_tile_v(hipStream_t st, const MixedArgs& a, const RowSrc<uint16_t>& gate) {
  if (a.dvp == 64) return launch_tile_heads<KS, 1, 4>(st, a, gate);
  if (a.dvp == 128) return launch_tile_heads<KS, 1, 8>(st, a, gate);
  return launch_tile_heads<KS, 2, 8>(st, a, gate);
}
template <int NH, int NJ, int HT>
int launch_value(hipStream_t st, const MixedArgs& a) {
  constexpr int GP = HT * 16;
  const size_t lds = (size_t)(2 * a.kv_chunk * (GP + 8) + GP * (a.kv_chunk + 8)) * 2;
  static std::once_flag once;
  static int rc = TNX_OK;
  std::call_once(once, [] { rc = raise_lds(&mixed_value_kernel<NH, NJ, HT>, (size_t)(2 * kMaxChunk * (GP + 8) + GP * (kMaxChunk + 8)) * 2); });
  if (rc) return rc;
  hipLaunchKernelGGL((mixed_value_kernel<NH, NJ, HT>), dim3((unsigned)a.n_chunks, (unsigned)a.B), dim3(256), lds, st, a);
  TNX_CHECK_LAUNCH("mixed_value");
  return TNX_OK;
}
template <int NH, int NJ>
int launch_value_heads(hipStream_t st, const MixedArgs& a) {
  if (a.H <= 16) return launch_value<NH, NJ, 1>(st, a);
  if (a.H <= 32) return launch_value<NH, NJ, 2>(st, a);
  return launch_value<NH, NJ, 4>(st, a);
}

constexpr size_t kAnyLds = 144 * 1024;
template <typename T>
int launch_any(hipStream_t st, const MixedArgs& a, const RowSrc<T>& gate) {
  const size_t lds = (size_t)a.H * (128 + 2 + a.dv) * 4;
  TNX_REQUIRE(lds <= kAnyLds, "mixed_attn: %d heads of %d values do not fit LDS", a.H, a.dv);
  static std::once_flag once;
  static int rc = TNX_OK;
  std::call_once(once, [] { rc = raise_lds(&mixed_any_kernel<T>, kAnyLds); });
  if (rc) return rc;
  hipLaunchKernelGGL((mixed_any_kernel<T>), dim3((unsigned)(a.B * a.T)), dim3(256), lds, st, a, gate);
  TNX_CHECK_LAUNCH("mixed_any");
  return TNX_OK;
}
bool mfma_size(int n) { return n == 64 || n == 128 || n == 256; }
int64_t score_row(int64_t S) { return cdiv(S, 64) * 64; }

}  // namespace

extern "C" int tnx_mixed_attn_ok(int64_t T, int64_t S, int H, int G, int dkp, int dvp) {
  if (T <= 0 || S <= 0 || H <= 0 || G <= 0 || H % G || !mfma_size(dkp) || !mfma_size(dvp)) return 0;
  if ((uint64_t)G * (uint64_t)S * (uint64_t)(dkp > dvp ? dkp : dvp) * 2 >= (1ull << 31)) return 0;
  if (T == 1) return H <= 64;
  return H <= (dkp <= 128 && dvp <= 128 ? 32 : 16);
}

extern "C" size_t tnx_mixed_attn_ws_bytes(int64_t B, int64_t T, int64_t S, int H, int dvp, int kv_chunk) {
  if (B <= 0 || T <= 0 || S <= 0 || H <= 0) return 0;
  if (T > 1) return (size_t)(B * T) * (size_t)H * 4;
  if (kv_chunk <= 0) return 0;
  return (size_t)(B * H) * ((size_t)score_row(S) + (size_t)cdiv(S, 64) * 2 + (size_t)cdiv(S, kv_chunk) * (size_t)dvp) * 4;
}

extern "C" int tnx_mixed_attn(void* stream, const tnx_mixed_attn_desc* d) {
  TNX_REQUIRE(d, "mixed_attn: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->T > 0 && d->S >= d->T && d->H > 0 && d->G > 0 && d->H % d->G == 0, "mixed_attn: bad shape");
  TNX_REQUIRE(d->dk > 0 && d->dv > 0 && d->dkp >= d->dk && d->dvp >= d->dv, "mixed_attn: bad head sizes");
  TNX_REQUIRE(d->q && d->kcache && d->vcache && d->talk && d->starts && d->col_ptr && d->out, "mixed_attn: null pointer");
  TNX_REQUIRE(d->out_ld >= (int64_t)d->H * d->dv && (d->gate.ld == 0 || src_given(d->gate)), "mixed_attn: short output rows or no gate rows");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "mixed_attn: bad dtype %d", d->dtype);
  TNX_REQUIRE(d->B <= 65535 && d->B * d->T < (int64_t)1 << 31 && d->S < (int64_t)1 << 31, "mixed_attn: too many rows");
  MixedArgs a;
  memset(&a, 0, sizeof(a));
  a.B = d->B; a.T = d->T; a.S = d->S; a.H = d->H; a.G = d->G; a.R = d->H / d->G; a.dk = d->dk; a.dv = d->dv; a.dkp = d->dkp; a.dvp = d->dvp;
  a.scale = d->scale; a.q = d->q; a.k = d->kcache; a.v = d->vcache; a.talk = d->talk; a.starts = d->starts; a.col_ptr = d->col_ptr;
  a.gated = d->gate.ld > 0; a.g_off = d->g_off; a.out = d->out; a.out_ld = d->out_ld; a.out_frag = d->out_frag;
  hipStream_t st = as_stream(stream);
  const RowSrc<uint16_t> g16{(const uint16_t*)d->gate.y, d->gate.ws, d->gate.split_k, d->gate.plane, d->gate.ld};
  const RowSrc<float> g32{(const float*)d->gate.y, d->gate.ws, d->gate.split_k, d->gate.plane, d->gate.ld};
  if (d->dtype == TNX_F32) return launch_any<float>(st, a, g32);
  if (!tnx_mixed_attn_ok(d->T, d->S, d->H, d->G, d->dkp, d->dvp)) return launch_any<uint16_t>(st, a, g16);
  TNX_REQUIRE(d->ws, "mixed_attn: needs the workspace of tnx_mixed_attn_ws_bytes");
  if (d->T > 1) {
    TNX_REQUIRE(d->G <= 65535 && cdiv(d->T, 16) <= 65535, "mixed_attn: too many kv heads or positions");
    a.lse = d->ws;
    switch (d->dkp) {
      case 64: return launch_tile_v<2>(st, a, g16);
      case 128: return launch_tile_v<4>(st, a, g16);
      default: return launch_tile_v<8>(st, a, g16);
    }
  }
  TNX_REQUIRE(d->kv_chunk > 0 && d->kv_chunk % 64 == 0 && d->kv_chunk <= kMaxChunk, "mixed_attn: kv_chunk must be a multiple of 64 up to %d", kMaxChunk);
  a.kv_chunk = d->kv_chunk;
  a.n_chunks = (int)cdiv(d->S, d->kv_chunk);
  a.Sp = score_row(d->S);
  // a wave of the score kernel takes as many keys as leave one or two waves per SIMD
  const int64_t streams = d->B * d->G * cdiv(a.R, 16), most = cdiv(d->S, 64), want = cdiv(1536, streams);
  a.s_chunk = (int)(cdiv(most, want < most ? want : most) * 64);
  a.s_chunks = (int)cdiv(d->S, a.s_chunk);
  a.scores = d->ws;
  a.ml = a.scores + d->B * d->H * a.Sp;
  a.part = a.ml + d->B * d->H * most * 2;
  const dim3 sg((unsigned)a.s_chunks, (unsigned)(d->G * cdiv(a.R, 16)), (unsigned)d->B);
  TNX_REQUIRE(sg.y <= 65535, "mixed_attn: too many heads");
  switch (d->dkp) {
    case 64: hipLaunchKernelGGL(mixed_score_kernel<2>, sg, dim3(64), 0, st, a); break;
    case 128: hipLaunchKernelGGL(mixed_score_kernel<4>, sg, dim3(64), 0, st, a); break;
    default: hipLaunchKernelGGL(mixed_score_kernel<8>, sg, dim3(64), 0, st, a); break;
  }
  TNX_CHECK_LAUNCH("mixed_score");
  const int rc = d->dvp == 64 ? launch_value_heads<1, 4>(st, a) : d->dvp == 128 ? launch_value_heads<1, 8>(st, a) : launch_value_heads<2, 8>(st, a);
  if (rc) return rc;
  const int64_t items = cdiv((int64_t)d->H * d->dv, 256);
  hipLaunchKernelGGL(mixed_join_kernel, dim3((unsigned)d->B, (unsigned)(items < 64 ? items : 64)), dim3(256), 0, st, a, g16);
  TNX_CHECK_LAUNCH("mixed_join");
  return TNX_OK;
}
