// Attention through a latent: a position's keys and values of all heads are linear in one normed vector
// c [rank], beside which one rotated key part [rot] is shared by the heads.  The cache holds a row
//   [c, zeros to rank_pad | rotated key part | zeros to row]
// per position.  Two ways to use it:
//   * prompts: c is expanded to per-head keys and values, and the query rows run through tnx_sink_attn
//     (latent_q_kernel, latent_kv_kernel lay its operands out);
//   * decoding and portions: the key projection is applied to the query instead, so that all heads attend
//     to the cache rows themselves (latent_attn_kernel: scores over the whole row, values its first `rank`
//     columns), and the value projection to the result.
// Norms, angles, scores and softmax are fp32.
#include <string.h>

#include <mutex>

#include "decoder.h"
#include "gemm_tile.h"

namespace {

constexpr float kNegBig = -1.0e30f;
constexpr float kLog2e = 1.4426950408889634f;
__device__ __forceinline__ float exp2_hw(float x) { return __builtin_amdgcn_exp2f(x); }

// ---- norms of the two latents, rotation of the shared key part, cache write ----------------------
struct LatentPrepArgs {
  int64_t T, S;
  int q_rank, rank, rot, rank_pad, row;
  float eps;
  int64_t q_off, kv_off;
  const float* w_q;
  const float* w_kv;
  const float* inv_freq;
  const int32_t* starts;
  const int32_t* col_ptr;
  int64_t q_ld, c_ld;
  int q_frag, c_frag;
};

template <typename T>
__global__ __launch_bounds__(256) void latent_prep_kernel(const LatentPrepArgs a, const RowSrc<T> src, T* q_out, T* c_out, T* cache) {
  extern __shared__ __align__(16) float sm[];   // query latent, key / value latent, rotated part
  __shared__ float red[2][4];
  const int64_t row = blockIdx.x, b = row / a.T, t = row % a.T;
  const int slot = *a.col_ptr + (int)t, tid = threadIdx.x;
  if (slot >= a.S) return;                                    // (uniform; the host sizes the cache)
  float sq = 0.f, skv = 0.f;
  for (int i = tid; i < a.q_rank; i += 256) {
    const float v = src.get(row, a.q_off + i);
    sm[i] = v;
    sq += v * v;
  }
  for (int i = tid; i < a.rank + a.rot; i += 256) {
    const float v = src.get(row, a.kv_off + i);
    sm[a.q_rank + i] = v;
    if (i < a.rank) skv += v * v;
  }
  sq = wave_sum(sq);
  skv = wave_sum(skv);
  if ((tid & 63) == 0) {
    red[0][tid >> 6] = sq;
    red[1][tid >> 6] = skv;
  }
  __syncthreads();
  const float rq = 1.0f / sqrtf((red[0][0] + red[0][1] + red[0][2] + red[0][3]) / (float)a.q_rank + a.eps);
  const float rkv = 1.0f / sqrtf((red[1][0] + red[1][1] + red[1][2] + red[1][3]) / (float)a.rank + a.eps);
  for (int i = tid; i < a.q_rank; i += 256)
    st_elem(q_out, a.q_frag ? frag_index(row, i, a.q_ld) : row * a.q_ld + i, sm[i] * rq * a.w_q[i]);
  T* dst = cache + (b * a.S + slot) * a.row;
  const float* kv = sm + a.q_rank;
  const float pos = (float)max(slot - a.starts[b], 0);
  for (int i = tid; i < a.row; i += 256) {
    float v = 0.f;
    if (i < a.rank) {
      v = kv[i] * rkv * a.w_kv[i];
      if (c_out) st_elem(c_out, a.c_frag ? frag_index(row, i, a.c_ld) : row * a.c_ld + i, v);
    } else if (i >= a.rank_pad && i < a.rank_pad + a.rot) {
      const int j = i - a.rank_pad;
      float sn, cs;
      sincosf(pos * a.inv_freq[j >> 1], &sn, &cs);
      const float u = kv[a.rank + (j & ~1)], w = kv[a.rank + (j | 1)];
      v = (j & 1) ? w * cs + u * sn : u * cs - w * sn;
    }
    st_elem(dst, i, v);
  }
}

// Latents, offsets and rows in whole runs of eight: a thread keeps its runs in registers.
template <int MAXI, typename T>
__global__ __launch_bounds__(256) void latent_prep_vec_kernel(const LatentPrepArgs a, const RowSrc<T> src, T* q_out, T* c_out, T* cache) {
  __shared__ float red[2][4];
  const int64_t row = blockIdx.x, b = row / a.T, t = row % a.T;
  const int slot = *a.col_ptr + (int)t, tid = threadIdx.x;
  if (slot >= a.S) return;                                    // (uniform)
  const int nq = a.q_rank / 8, nkv = a.rank / 8, nr = a.rot / 8, n = nq + nkv + nr;
  float f[MAXI][8], w[MAXI][8];
  const RowSrc<float> wq{a.w_q, nullptr, 1, 0, 0}, wkv{a.w_kv, nullptr, 1, 0, 0};
#pragma unroll
  for (int c = 0; c < MAXI; ++c) {
    const int i = min(c * 256 + tid, n - 1);
    get8(src, row, i < nq ? a.q_off + i * 8 : a.kv_off + (i - nq) * 8, f[c]);
    if (i < nq) get8(wq, 0, i * 8, w[c]);
    else if (i < nq + nkv) get8(wkv, 0, (i - nq) * 8, w[c]);
  }
  const float pos = (float)max(slot - a.starts[b], 0);
  float sq = 0.f, skv = 0.f;
#pragma unroll
  for (int c = 0; c < MAXI; ++c) {
    const int i = c * 256 + tid;
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) s += f[c][j] * f[c][j];
    if (i < nq) sq += s;
    else if (i < nq + nkv) skv += s;
  }
  sq = wave_sum(sq);
  skv = wave_sum(skv);
  if ((tid & 63) == 0) {
    red[0][tid >> 6] = sq;
    red[1][tid >> 6] = skv;
  }
  __syncthreads();
  const float rq = 1.0f / sqrtf((red[0][0] + red[0][1] + red[0][2] + red[0][3]) / (float)a.q_rank + a.eps);
  const float rkv = 1.0f / sqrtf((red[1][0] + red[1][1] + red[1][2] + red[1][3]) / (float)a.rank + a.eps);
  T* dst = cache + (b * a.S + slot) * a.row;
#pragma unroll
  for (int c = 0; c < MAXI; ++c) {
    const int i = c * 256 + tid;
    if (i >= n) continue;
    if (i < nq + nkv) {
      const float r = i < nq ? rq : rkv;
#pragma unroll
      for (int j = 0; j < 8; ++j) f[c][j] = f[c][j] * r * w[c][j];
      if (i < nq) {
        put8(q_out + (a.q_frag ? frag_index(row, i * 8, a.q_ld) : row * a.q_ld + i * 8), f[c]);
      } else {
        const int d = (i - nq) * 8;
        put8(dst + d, f[c]);
        if (c_out) put8(c_out + (a.c_frag ? frag_index(row, d, a.c_ld) : row * a.c_ld + d), f[c]);
      }
      continue;
    }
    const int j0 = (i - nq - nkv) * 8;
    float o[8];
#pragma unroll
    for (int p = 0; p < 4; ++p) {
      float sn, cs;
      sincosf(pos * a.inv_freq[j0 / 2 + p], &sn, &cs);
      o[2 * p] = f[c][2 * p] * cs - f[c][2 * p + 1] * sn;
      o[2 * p + 1] = f[c][2 * p + 1] * cs + f[c][2 * p] * sn;
    }
    put8(dst + a.rank_pad + j0, o);
  }
  for (int i = a.rank + tid; i < a.row; i += 256)
    if (i < a.rank_pad || i >= a.rank_pad + a.rot) st_elem(dst, i, 0.f);
}

// ---- queries: the unrotated part of every head to one place, the rotated part to another ----------
struct LatentQArgs {
  int64_t T;
  int H, n, r;
  const float* inv_freq;
  const int32_t* starts;
  const int32_t* col_ptr;
  int64_t un_ld, rot_ld;   // stride of a head
  int un_pad, rot_pad;     // elements written of a head (zeros behind n / r)
};
constexpr int kMaxPairs = 512;

template <typename T>
__global__ __launch_bounds__(256) void latent_q_kernel(const LatentQArgs a, const RowSrc<T> src, T* un, T* rot) {
  __shared__ float sn[kMaxPairs], cs[kMaxPairs];
  const int64_t row = blockIdx.x, b = row / a.T, t = row % a.T;
  const float pos = (float)max(*a.col_ptr + (int)t - a.starts[b], 0);
  for (int i = threadIdx.x; i < a.r / 2; i += 256) sincosf(pos * a.inv_freq[i], &sn[i], &cs[i]);
  __syncthreads();
  const int per = a.un_pad + a.rot_pad, d = a.n + a.r;
  for (int it = threadIdx.x; it < a.H * per; it += 256) {
    const int h = it / per, i = it % per;
    if (i < a.un_pad) {
      st_elem(un, (row * a.H + h) * a.un_ld + i, i < a.n ? src.get(row, (int64_t)h * d + i) : 0.f);
      continue;
    }
    const int j = i - a.un_pad;
    float v = 0.f;
    if (j < a.r) {
      const float u = src.get(row, (int64_t)h * d + a.n + (j & ~1)), w = src.get(row, (int64_t)h * d + a.n + (j | 1));
      v = (j & 1) ? w * cs[j >> 1] + u * sn[j >> 1] : u * cs[j >> 1] - w * sn[j >> 1];
    }
    st_elem(rot, (row * a.H + h) * a.rot_ld + j, v);
  }
}
// everything in whole runs of eight; the items of a row are spread over gridDim.y work-groups
template <typename T>
__global__ __launch_bounds__(256) void latent_q_vec_kernel(const LatentQArgs a, const RowSrc<T> src, T* un, T* rot) {
  __shared__ float sn[kMaxPairs], cs[kMaxPairs];
  const int64_t row = blockIdx.x, b = row / a.T, t = row % a.T;
  const float pos = (float)max(*a.col_ptr + (int)t - a.starts[b], 0);
  for (int i = threadIdx.x; i < a.r / 2; i += 256) sincosf(pos * a.inv_freq[i], &sn[i], &cs[i]);
  __syncthreads();
  const int un8 = a.un_pad / 8, per = un8 + a.rot_pad / 8, d = a.n + a.r;
  for (int it = blockIdx.y * 256 + threadIdx.x; it < a.H * per; it += 256 * gridDim.y) {
    const int h = it / per, i = it % per;
    float f[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) f[j] = 0.f;
    if (i < un8) {
      if (i * 8 < a.n) get8(src, row, (int64_t)h * d + i * 8, f);
      put8(un + (row * a.H + h) * a.un_ld + i * 8, f);
      continue;
    }
    const int j0 = (i - un8) * 8;
    if (j0 < a.r) {
      float u[8];
      get8(src, row, (int64_t)h * d + a.n + j0, u);
#pragma unroll
      for (int p = 0; p < 4; ++p) {
        const float co = cs[j0 / 2 + p], si = sn[j0 / 2 + p];
        f[2 * p] = u[2 * p] * co - u[2 * p + 1] * si;
        f[2 * p + 1] = u[2 * p + 1] * co + u[2 * p] * si;
      }
    }
    put8(rot + (row * a.H + h) * a.rot_ld + j0, f);
  }
}

// ---- expanded keys and values of a prompt ---------------------------------------------------------
struct LatentKvArgs {
  int64_t T, S;            // tokens of a row of k and v; columns of the cache
  int H, n, r, vd, dkp, dvp, rank_pad, row;
  int64_t v_off;
};
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void latent_kv_kernel(const LatentKvArgs a, const RowSrc<T> src, const T* cache, T* k, T* v) {
  const int64_t row = blockIdx.x, b = row / a.T, t = row % a.T;
  const T* rot = cache + (b * a.S + t) * a.row + a.rank_pad;
  constexpr int W = VEC ? 8 : 1;
  const int kc = a.dkp / W, per = kc + a.dvp / W;
  for (int it = blockIdx.y * 256 + threadIdx.x; it < a.H * per; it += 256 * gridDim.y) {
    const int h = it / per, i = it % per;
    const bool is_k = i < kc;
    const int d = (is_k ? i : i - kc) * W;
    T* dst = is_k ? k + ((b * a.H + h) * a.T + t) * a.dkp + d : v + ((b * a.H + h) * a.T + t) * a.dvp + d;
    if constexpr (VEC) {
      float f[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) f[j] = 0.f;
      if (is_k) {
        if (d < a.n) get8(src, row, (int64_t)h * a.n + d, f);
        else if (d < a.n + a.r) get8(RowSrc<T>{rot, nullptr, 1, 0, 0}, 0, d - a.n, f);
      } else if (d < a.vd) {
        get8(src, row, a.v_off + (int64_t)h * a.vd + d, f);
      }
      put8(dst, f);
    } else {
      float f = 0.f;
      if (is_k) {
        if (d < a.n) f = src.get(row, (int64_t)h * a.n + d);
        else if (d < a.n + a.r) f = ld_elem(rot, d - a.n);
      } else if (d < a.vd) {
        f = src.get(row, a.v_off + (int64_t)h * a.vd + d);
      }
      st_elem(dst, 0, f);
    }
  }
}

// ---- attention of all heads to the cache rows -----------------------------------------------------
struct LatentAttnArgs {
  int64_t B, T, S;
  int H, rank;
  float scale;
  const uint16_t* q;       // [B * T, H, row]
  const uint16_t* cache;   // [B, S, row]
  const int32_t* starts;
  const int32_t* col_ptr;
  int kv_chunk, n_chunks;
  float* ws;
  uint16_t* out;           // [B * T, H, out_head]
  int64_t out_head;
};

constexpr int kKeys = 64;
constexpr size_t latent_smem_bytes(int ks) {
  return (size_t)(2 * kKeys * ks * 32 + 32 * (kKeys + 8)) * 2 + 2 * 4 * 32 * 4;
}

// 32 query rows ((position, head) pairs, heads fastest) per work-group; 64 cache rows at a time in LDS, where
// they serve the scores as keys and the output as values, while the next 64 are on their way into the other
// buffer.  Wave w of eight forms the scores of keys 16 (w % 4) .. + 15 with one half of the queries and the output's
// columns 16 NV w .. + 16 NV - 1 for all of them; both products are transposed, so that a lane owns one query.
// The 16-byte chunks of a row are permuted within groups of eight (by the row's number), so that neither the 16
// rows of a score fragment nor the columns of a value row meet in a bank.
template <int KS, int NV>   // 32-deep k-steps of a row; 128-column groups of the values
__global__ __launch_bounds__(512) __attribute__((amdgpu_waves_per_eu(2, 2))) void latent_attn_kernel(const LatentAttnArgs a) {
  constexpr int LP = KS * 32, DV = NV * 128, PLD = kKeys + 8, CH = LP / 8, CW = NV / 2;   // CW: 32-column groups per wave
  constexpr int PIECES = KS / 2;
  constexpr uint32_t kBuf = kKeys * LP * 2;
  constexpr bool kHalfStride = LP / 2 % 64 == 32;           // rows alternate between the halves of the banks
  extern __shared__ __align__(16) unsigned char smem[];
  uint16_t* ps = reinterpret_cast<uint16_t*>(smem + 2 * kBuf);
  float* redm = reinterpret_cast<float*>(ps + 32 * PLD);    // [4][32]
  float* redl = redm + 128;
  const int tid = threadIdx.x, lane = tid & 63, l32 = lane & 31, lh = lane >> 5, lm = lane & 15, lq = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), kg = wave & 3, half = wave >> 2;
  const int chunk = blockIdx.x, tile = blockIdx.y;
  const int64_t b = blockIdx.z;
  const int col0 = *a.col_ptr, start = a.starts[b];
  const unsigned rows = (unsigned)(a.T * a.H);
  int k_lo = max(start, 0), k_hi = min(col0 + (int)(min((unsigned)tile * 32 + 31, rows - 1) / a.H), (int)a.S - 1);
  if (a.n_chunks > 1) {
    k_lo = max(k_lo, chunk * a.kv_chunk);
    k_hi = min(k_hi, chunk * a.kv_chunk + a.kv_chunk - 1);
  }
  auto swz = [](int row) { return kHalfStride ? (row >> 1) & 7 : row & 7; };
  // cache rows -> LDS: piece c of this wave is one kilobyte
  const u32x4 rk = raw_rsrc(a.cache + b * a.S * LP, (uint64_t)a.S * LP * 2);
  const uint32_t lds0 = lds_addr(smem) + (uint32_t)wave * (PIECES * 1024u);
  uint32_t off[PIECES];
#pragma unroll
  for (int c = 0; c < PIECES; ++c) {
    const int g = (wave * PIECES + c) * 64 + lane, row = g / CH, pc = g % CH;
    off[c] = (uint32_t)(row * (LP * 2) + ((pc & ~7) | ((pc ^ swz(row)) & 7)) * 16);
  }
  auto fetch = [&](int kb, uint32_t buf) {
#pragma unroll
    for (int c = 0; c < PIECES; ++c) dma16(lds0 + buf + (uint32_t)c * 1024u, rk, off[c] + (uint32_t)kb * (LP * 2), 0);
  };
  const int kb0 = k_lo & ~(kKeys - 1);
  if (kb0 <= k_hi) fetch(kb0, 0);
  const int hq = half * 16 + lm;                            // this lane's query in the scores
  const unsigned sq = min((unsigned)tile * 32 + hq, rows - 1);
  u32x4 qf[KS];
#pragma unroll
  for (int j = 0; j < KS; ++j)
    qf[j] = *reinterpret_cast<const u32x4*>(a.q + ((b * a.T + sq / a.H) * a.H + sq % a.H) * LP + lq * 8 + j * 32);
  const int cn = min(col0 + (int)(sq / a.H), k_hi);
  float m16 = kNegBig, l16 = 0.f, m32 = kNegBig;
  f32x16 O[CW];
#pragma unroll
  for (int j = 0; j < CW; ++j)
#pragma unroll
    for (int i = 0; i < 16; ++i) O[j][i] = 0.f;
  const float sc2 = a.scale * kLog2e;
  // this lane's score fragment: row 16 kg + lm, chunk 4 j + lq; its value columns: CW from vcol on
  const int krow = kg * 16 + lm, vcol = wave * (CW * 32) + l32 * CW, vch = vcol / 8;
  const uint32_t kf0 = (uint32_t)(krow * (LP * 2) + ((lq ^ swz(krow)) & 7) * 16), kf1 = (uint32_t)(krow * (LP * 2) + (((4 + lq) ^ swz(krow)) & 7) * 16);
  uint32_t buf = 0;
  for (int kb = kb0; kb <= k_hi; kb += kKeys, buf ^= kBuf) {
    tnx_wait_vm(0);
    __syncthreads();            // these rows have landed; every wave is done with the other buffer
    if (kb + kKeys <= k_hi) fetch(kb + kKeys, buf ^ kBuf);
    const unsigned char* ks = smem + buf;
    f32x4 st[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};   // even and odd k-steps
    constexpr int PF = 4;
    u32x4 kf[PF];
    auto load_k = [&](int j) { kf[j % PF] = *reinterpret_cast<const u32x4*>(ks + ((j & 1) ? kf1 : kf0) + (j >> 1) * 128); };
#pragma unroll
    for (int j = 0; j < PF && j < KS; ++j) load_k(j);
#pragma unroll
    for (int j = 0; j < KS; ++j) {
      st[j & 1] = mfma16(kf[j % PF], qf[j], st[j & 1]);
      if (j + PF < KS) load_k(j + PF);
      __builtin_amdgcn_sched_barrier(0);
    }
    // register i: key kb + 16 kg + 4 lq + i
    float sc[4], mx = -__builtin_inff();
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int key = kb + kg * 16 + 4 * lq + i;
      sc[i] = key >= k_lo && key <= cn ? (st[0][i] + st[1][i]) * sc2 : -__builtin_inff();
      mx = fmaxf(mx, sc[i]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    if (lq == 0) redm[kg * 32 + hq] = mx;
    __syncthreads();
    {
      const float m_new = fmaxf(m16, fmaxf(fmaxf(redm[hq], redm[32 + hq]), fmaxf(redm[64 + hq], redm[96 + hq])));
      float p[4], psum = 0.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        p[i] = exp2_hw(sc[i] - m_new);   // (exp2(-inf) = 0: a masked key)
        psum += p[i];
      }
      *reinterpret_cast<u32x2*>(&ps[hq * PLD + kg * 16 + 4 * lq]) = u32x2{pack2bf(p[0], p[1]), pack2bf(p[2], p[3])};
      l16 = l16 * exp2_hw(m16 - m_new) + psum;
      m16 = m_new;
    }
    const float m_new = fmaxf(m32, fmaxf(fmaxf(redm[l32], redm[32 + l32]), fmaxf(redm[64 + l32], redm[96 + l32])));
    const float alpha = exp2_hw(m32 - m_new);
    m32 = m_new;
    if (__builtin_amdgcn_ballot_w64(alpha != 1.0f) != 0) {
#pragma unroll
      for (int j = 0; j < CW; ++j)
#pragma unroll
        for (int i = 0; i < 16; ++i) O[j][i] *= alpha;
    }
    uint32_t v[2][8];
    u32x4 pf[2];
    auto load_v = [&](int s) {
      // k index 8 lh + i of this step: key 16 s + 8 lh + i
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int row = 16 * s + 8 * lh + i;
        const unsigned char* at = ks + row * (LP * 2) + ((vch & ~7) | ((vch ^ swz(row)) & 7)) * 16 + vcol % 8 * 2;
        if constexpr (CW == 2) v[s & 1][i] = *reinterpret_cast<const uint32_t*>(at);
        else v[s & 1][i] = *reinterpret_cast<const uint16_t*>(at);
      }
    };
    load_v(0);
    __syncthreads();
    auto load_p = [&](int s) { pf[s & 1] = *reinterpret_cast<const u32x4*>(&ps[l32 * PLD + 16 * s + 8 * lh]); };
    load_p(0);
#pragma unroll
    for (int s = 0; s < kKeys / 16; ++s) {
      if (s + 1 < kKeys / 16) {
        load_v(s + 1);
        load_p(s + 1);
      }
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int j = 0; j < CW; ++j) {
        const uint32_t sel = j ? 0x07060302u : 0x05040100u;
        u32x4 af;
#pragma unroll
        for (int r = 0; r < 4; ++r) af[r] = __builtin_amdgcn_perm(v[s & 1][2 * r + 1], v[s & 1][2 * r], sel);
        O[j] = mfma32(af, pf[s & 1], O[j]);
      }
    }
  }
  l16 += __shfl_xor(l16, 16, 64);
  l16 += __shfl_xor(l16, 32, 64);
  if (lq == 0) redl[kg * 32 + hq] = l16;
  __syncthreads();
  const float l = redl[l32] + redl[32 + l32] + redl[64 + l32] + redl[96 + l32];
  const unsigned qrow = (unsigned)tile * 32 + l32;
  if (qrow >= rows) return;
  const int64_t qv = (b * a.T + qrow / a.H) * a.H + qrow % a.H;
  // register 4 b + e of O[j]: column 32 CW wave + CW (8 b + 4 lh + e) + j: runs of 4 CW columns
  const float w = a.n_chunks > 1 ? 1.0f : l > 0.f ? 1.0f / l : 0.f;
#pragma unroll
  for (int bb = 0; bb < 4; ++bb) {
    const int d0 = wave * (CW * 32) + CW * (8 * bb + 4 * lh);
    float x[4 * CW];
#pragma unroll
    for (int e = 0; e < 4; ++e)
#pragma unroll
      for (int j = 0; j < CW; ++j) x[e * CW + j] = O[j][4 * bb + e] * w;
    if (a.n_chunks > 1) {
      float* po = a.ws + (qv * a.n_chunks + chunk) * DV + d0;
#pragma unroll
      for (int c = 0; c < 4 * CW; c += 4) *reinterpret_cast<f32x4*>(po + c) = f32x4{x[c], x[c + 1], x[c + 2], x[c + 3]};
      continue;
    }
    uint16_t* out = a.out + qv * a.out_head + d0;
#pragma unroll
    for (int c = 0; c < 4 * CW; c += 4) {
      if (d0 + c + 4 <= a.rank) {
        *reinterpret_cast<u32x2*>(out + c) = u32x2{pack2bf(x[c], x[c + 1]), pack2bf(x[c + 2], x[c + 3])};
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (d0 + c + e < a.rank) out[c + e] = f2bf(x[c + e]);
      }
    }
  }
  if (a.n_chunks > 1 && wave == 0 && lh == 0) {
    float* ml = a.ws + a.B * a.T * a.H * a.n_chunks * DV + (qv * a.n_chunks + chunk) * 2;
    ml[0] = m32;
    ml[1] = l;
  }
}

// one work-group per query vector: merges the chunks
__global__ __launch_bounds__(128) void latent_merge_kernel(const LatentAttnArgs a, int dv) {
  extern __shared__ float wts[];   // [n_chunks]
  __shared__ float tot;
  const int64_t qv = blockIdx.x;
  const float* ml = a.ws + a.B * a.T * a.H * a.n_chunks * dv + qv * a.n_chunks * 2;
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
    if (threadIdx.x == 0) tot = l > 0.f ? 1.0f / l : 0.f;
  }
  __syncthreads();
  const float* po = a.ws + qv * a.n_chunks * dv;
  for (int d = threadIdx.x * 4; d < a.rank; d += 512) {
    f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int c = 0; c < a.n_chunks; ++c)
      if (wts[c] != 0.f) acc += wts[c] * *reinterpret_cast<const f32x4*>(po + (int64_t)c * dv + d);
    uint16_t* out = a.out + qv * a.out_head + d;
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (d + e < a.rank) out[e] = f2bf(acc[e] * tot);
  }
}

template <int KS, int NV>
int launch_latent(hipStream_t st, const LatentAttnArgs& a) {
  static std::once_flag once;
  static hipError_t e = hipSuccess;
  constexpr size_t kSmem = latent_smem_bytes(KS);
  static_assert(kSmem <= 160 * 1024, "the tile fits LDS");
  std::call_once(once, [] {
    e = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_attn_kernel<KS, NV>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kSmem);
  });
  if (e != hipSuccess) {
    tnx_set_error("latent_attn: cannot raise the dynamic LDS limit: %s", hipGetErrorString(e));
    return TNX_ELAUNCH;
  }
  hipLaunchKernelGGL((latent_attn_kernel<KS, NV>), dim3((unsigned)a.n_chunks, (unsigned)cdiv(a.T * a.H, 32), (unsigned)a.B), dim3(512), kSmem, st, a);
  if (a.n_chunks > 1)
    hipLaunchKernelGGL(latent_merge_kernel, dim3((unsigned)(a.B * a.T * a.H)), dim3(128), (size_t)a.n_chunks * 4, st, a, NV * 128);
  TNX_CHECK_LAUNCH("latent_attn");
  return TNX_OK;
}

// ---- y * sigmoid(gate) ----------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void gate_mul_kernel(const T* y, int64_t y_ld, int head, int64_t y_head, const RowSrc<T> g, int64_t g_off,
                                                       int64_t W, T* out, int64_t out_ld, int out_frag) {
  const int64_t row = blockIdx.x;
  for (int64_t i = (int64_t)blockIdx.y * 256 + threadIdx.x; i < W; i += 256 * gridDim.y)
    st_elem(out, out_frag ? frag_index(row, i, out_ld) : row * out_ld + i,
            ld_elem(y, row * y_ld + i / head * y_head + i % head) * sigmoid_f32(g.get(row, g_off + i)));
}
template <typename T>
__global__ __launch_bounds__(256) void gate_mul_vec_kernel(const T* y, int64_t y_ld, int head, int64_t y_head, const RowSrc<T> g, int64_t g_off,
                                                           int64_t W, T* out, int64_t out_ld, int out_frag) {
  const int64_t row = blockIdx.x;
  const RowSrc<T> ys{y, nullptr, 1, 0, y_ld};
  for (int64_t i = ((int64_t)blockIdx.y * 256 + threadIdx.x) * 8; i < W; i += 2048 * gridDim.y) {
    float v[8], z[8];
    get8(ys, row, i / head * y_head + i % head, v);
    get8(g, row, g_off + i, z);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] *= sigmoid_f32(z[j]);
    put8(out + (out_frag ? frag_index(row, i, out_ld) : row * out_ld + i), v);
  }
}

template <typename T>
RowSrc<T> row_src(const tnx_rows_src& s) {
  return RowSrc<T>{reinterpret_cast<const T*>(s.y), s.ws, s.split_k, s.plane, s.ld};
}
// work-groups of a row: few rows spread their items, many rows fill the device by themselves
unsigned spread(int64_t rows, int64_t items) {
  if (rows >= 1024) return 1;
  const int64_t n = cdiv(items, 256);
  return (unsigned)(n < 64 ? n : 64);
}
template <typename T>
int prep_launch(hipStream_t st, const tnx_latent_prep_desc* d, const LatentPrepArgs& a) {
  const size_t lds = (size_t)(d->q_rank + d->rank + d->rot) * 4;
  const int items = (d->q_rank + d->rank + d->rot) / 8;
  const bool vec = (d->q_rank | d->rank | d->rot | d->row) % 8 == 0 && d->q_off % 8 == 0 && d->kv_off % 8 == 0 && d->y.ld % 8 == 0 &&
                   d->y.plane % 8 == 0 && d->q_ld % 8 == 0 && d->c_ld % 8 == 0 && items <= 1024;
  const dim3 grid((unsigned)(d->B * d->T));
  T *q_out = (T*)d->q_out, *c_out = (T*)d->c_out, *cache = (T*)d->cache;
  if (vec && items <= 256) hipLaunchKernelGGL((latent_prep_vec_kernel<1, T>), grid, dim3(256), 0, st, a, row_src<T>(d->y), q_out, c_out, cache);
  else if (vec && items <= 512) hipLaunchKernelGGL((latent_prep_vec_kernel<2, T>), grid, dim3(256), 0, st, a, row_src<T>(d->y), q_out, c_out, cache);
  else if (vec) hipLaunchKernelGGL((latent_prep_vec_kernel<4, T>), grid, dim3(256), 0, st, a, row_src<T>(d->y), q_out, c_out, cache);
  else hipLaunchKernelGGL(latent_prep_kernel<T>, grid, dim3(256), lds, st, a, row_src<T>(d->y), q_out, c_out, cache);
  TNX_CHECK_LAUNCH("latent_prep");
  return TNX_OK;
}
template <typename T>
int q_launch(hipStream_t st, const tnx_latent_q_desc* d, const LatentQArgs& a) {
  const bool vec = (d->n | d->r | d->un_pad | d->rot_pad) % 8 == 0 && d->un_ld % 8 == 0 && d->rot_ld % 8 == 0 && d->y.ld % 8 == 0 &&
                   d->y.plane % 8 == 0 && ((uintptr_t)d->un & 15) == 0 && ((uintptr_t)d->rot & 15) == 0;
  const int64_t M = d->B * d->T;
  if (vec)
    hipLaunchKernelGGL(latent_q_vec_kernel<T>, dim3((unsigned)M, spread(M, (int64_t)d->H * (d->un_pad + d->rot_pad) / 8)), dim3(256), 0, st, a,
                       row_src<T>(d->y), (T*)d->un, (T*)d->rot);
  else
    hipLaunchKernelGGL(latent_q_kernel<T>, dim3((unsigned)M), dim3(256), 0, st, a, row_src<T>(d->y), (T*)d->un, (T*)d->rot);
  TNX_CHECK_LAUNCH("latent_q");
  return TNX_OK;
}
template <typename T>
int kv_launch(hipStream_t st, const tnx_latent_kv_desc* d, const LatentKvArgs& a) {
  const bool vec = (d->n | d->r | d->vd | d->dkp | d->dvp | d->rank_pad | d->row) % 8 == 0 && d->v_off % 8 == 0 && d->y.ld % 8 == 0 && d->y.plane % 8 == 0;
  const int64_t M = d->B * d->T;
  if (vec)
    hipLaunchKernelGGL((latent_kv_kernel<T, true>), dim3((unsigned)M, spread(M, (int64_t)d->H * (d->dkp + d->dvp) / 8)), dim3(256), 0, st, a,
                       row_src<T>(d->y), (const T*)d->cache, (T*)d->k, (T*)d->v);
  else
    hipLaunchKernelGGL((latent_kv_kernel<T, false>), dim3((unsigned)M, spread(M, (int64_t)d->H * (d->dkp + d->dvp))), dim3(256), 0, st, a,
                       row_src<T>(d->y), (const T*)d->cache, (T*)d->k, (T*)d->v);
  TNX_CHECK_LAUNCH("latent_kv");
  return TNX_OK;
}
template <typename T>
int gate_launch(hipStream_t st, const tnx_gate_mul_desc* d) {
  const bool vec = d->head % 8 == 0 && d->y_head % 8 == 0 && d->y_ld % 8 == 0 && d->g_off % 8 == 0 && d->g.ld % 8 == 0 && d->g.plane % 8 == 0 &&
                   d->out_ld % 8 == 0;
  if (vec)
    hipLaunchKernelGGL(gate_mul_vec_kernel<T>, dim3((unsigned)d->M, spread(d->M, d->W / 8)), dim3(256), 0, st, (const T*)d->y, d->y_ld, d->head,
                       d->y_head, row_src<T>(d->g), d->g_off, d->W, (T*)d->out, d->out_ld, d->out_frag);
  else
    hipLaunchKernelGGL(gate_mul_kernel<T>, dim3((unsigned)d->M, spread(d->M, d->W)), dim3(256), 0, st, (const T*)d->y, d->y_ld, d->head, d->y_head,
                       row_src<T>(d->g), d->g_off, d->W, (T*)d->out, d->out_ld, d->out_frag);
  TNX_CHECK_LAUNCH("gate_mul");
  return TNX_OK;
}
bool known_dtype(int t) { return t == TNX_BF16 || t == TNX_F32; }

}  // namespace

extern "C" int tnx_latent_row(int rank, int rot, int dtype) {
  if (rank <= 0 || rot < 0) return 0;
  const int n = (rank + 15) / 16 * 16 + rot;
  if (dtype != TNX_BF16) return (n + 3) / 4 * 4;
  if (rank <= 256 && n <= 128) return 128;
  if (rank <= 256 && n <= 256) return 256;
  if (rank <= 256 && n <= 320) return 320;
  if (rank <= 512 && n <= 576) return 576;
  return (n + 7) / 8 * 8;
}

extern "C" int tnx_latent_attn_ok(int rank, int row, int64_t S) {
  return ((rank <= 256 && (row == 128 || row == 256 || row == 320)) || (rank <= 512 && row == 576)) && S > 0 && S * row * 2 < ((int64_t)1 << 31);
}

extern "C" int tnx_latent_prep(void* stream, const tnx_latent_prep_desc* d) {
  TNX_REQUIRE(d, "latent_prep: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->T > 0 && d->S > 0 && d->q_rank > 0 && d->rank > 0 && d->rot >= 0 && d->rot % 2 == 0, "latent_prep: bad shape");
  TNX_REQUIRE(d->rank_pad >= d->rank && d->row >= d->rank_pad + d->rot && d->q_ld >= d->q_rank && (!d->c_out || d->c_ld >= d->rank), "latent_prep: short rows");
  TNX_REQUIRE((int64_t)d->q_rank + d->rank + d->rot <= 16384, "latent_prep: latents above 16384");
  TNX_REQUIRE(src_given(d->y) && d->w_q && d->w_kv && (d->rot == 0 || d->inv_freq) && d->starts && d->col_ptr && d->q_out && d->cache, "latent_prep: null pointer");
  TNX_REQUIRE(known_dtype(d->dtype), "latent_prep: bad dtype %d", d->dtype);
  LatentPrepArgs a;
  a.T = d->T; a.S = d->S; a.q_rank = d->q_rank; a.rank = d->rank; a.rot = d->rot; a.rank_pad = d->rank_pad; a.row = d->row; a.eps = d->eps;
  a.q_off = d->q_off; a.kv_off = d->kv_off; a.w_q = d->w_q; a.w_kv = d->w_kv; a.inv_freq = d->inv_freq; a.starts = d->starts; a.col_ptr = d->col_ptr;
  a.q_ld = d->q_ld; a.c_ld = d->c_ld; a.q_frag = d->q_frag; a.c_frag = d->c_frag;
  return d->dtype == TNX_BF16 ? prep_launch<uint16_t>(as_stream(stream), d, a) : prep_launch<float>(as_stream(stream), d, a);
}

extern "C" int tnx_latent_q(void* stream, const tnx_latent_q_desc* d) {
  TNX_REQUIRE(d, "latent_q: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->T > 0 && d->H > 0 && d->n > 0 && d->r >= 0 && d->r % 2 == 0 && d->r / 2 <= kMaxPairs, "latent_q: bad shape");
  TNX_REQUIRE(d->un_pad >= d->n && d->rot_pad >= d->r && d->un_ld >= d->n && d->rot_ld >= d->r, "latent_q: short heads");
  TNX_REQUIRE(src_given(d->y) && (d->r == 0 || d->inv_freq) && d->starts && d->col_ptr && d->un && d->rot, "latent_q: null pointer");
  TNX_REQUIRE(known_dtype(d->dtype), "latent_q: bad dtype %d", d->dtype);
  LatentQArgs a;
  a.T = d->T; a.H = d->H; a.n = d->n; a.r = d->r; a.inv_freq = d->inv_freq; a.starts = d->starts; a.col_ptr = d->col_ptr;
  a.un_ld = d->un_ld; a.rot_ld = d->rot_ld; a.un_pad = d->un_pad; a.rot_pad = d->rot_pad;
  return d->dtype == TNX_BF16 ? q_launch<uint16_t>(as_stream(stream), d, a) : q_launch<float>(as_stream(stream), d, a);
}

extern "C" int tnx_latent_kv(void* stream, const tnx_latent_kv_desc* d) {
  TNX_REQUIRE(d, "latent_kv: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->T > 0 && d->S >= d->T && d->H > 0 && d->n > 0 && d->r >= 0 && d->vd > 0, "latent_kv: bad shape");
  TNX_REQUIRE(d->dkp >= d->n + d->r && d->dvp >= d->vd && d->row >= d->rank_pad + d->r && d->rank_pad >= 0, "latent_kv: short rows");
  TNX_REQUIRE(src_given(d->y) && d->cache && d->k && d->v, "latent_kv: null pointer");
  TNX_REQUIRE(known_dtype(d->dtype), "latent_kv: bad dtype %d", d->dtype);
  LatentKvArgs a;
  a.T = d->T; a.S = d->S; a.H = d->H; a.n = d->n; a.r = d->r; a.vd = d->vd; a.dkp = d->dkp; a.dvp = d->dvp; a.rank_pad = d->rank_pad; a.row = d->row;
  a.v_off = d->v_off;
  return d->dtype == TNX_BF16 ? kv_launch<uint16_t>(as_stream(stream), d, a) : kv_launch<float>(as_stream(stream), d, a);
}

extern "C" size_t tnx_latent_attn_ws_bytes(int64_t B, int64_t T, int64_t S, int H, int rank, int kv_chunk) {
  if (kv_chunk <= 0 || kv_chunk >= S) return 0;
  return (size_t)(B * T * H) * (size_t)cdiv(S, kv_chunk) * (size_t)((rank <= 256 ? 256 : 512) + 2) * sizeof(float);
}

extern "C" int tnx_latent_attn(void* stream, const tnx_latent_attn_desc* d) {
  TNX_REQUIRE(d, "latent_attn: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->B <= 65535 && d->T > 0 && d->S >= d->T && d->H > 0 && d->rank > 0, "latent_attn: bad shape");
  TNX_REQUIRE(tnx_latent_attn_ok(d->rank, d->row, d->S), "latent_attn: no kernel for rank %d in rows of %d", d->rank, d->row);
  TNX_REQUIRE(d->q && d->cache && d->starts && d->col_ptr && d->out && d->out_head >= d->rank && d->out_head % 8 == 0, "latent_attn: null pointer or bad output heads");
  TNX_REQUIRE(cdiv(d->T * d->H, 32) <= 65535, "latent_attn: too many query tiles");
  LatentAttnArgs a;
  a.B = d->B; a.T = d->T; a.S = d->S; a.H = d->H; a.rank = d->rank; a.scale = d->scale; a.q = (const uint16_t*)d->q; a.cache = (const uint16_t*)d->cache;
  a.starts = d->starts; a.col_ptr = d->col_ptr; a.kv_chunk = d->kv_chunk; a.ws = d->ws; a.out = (uint16_t*)d->out; a.out_head = d->out_head;
  a.n_chunks = d->kv_chunk > 0 && d->kv_chunk < d->S ? (int)cdiv(d->S, d->kv_chunk) : 1;
  TNX_REQUIRE(a.n_chunks == 1 || (d->ws && d->kv_chunk % kKeys == 0), "latent_attn: a split key range needs a workspace and chunks of whole 64 keys");
  hipStream_t st = as_stream(stream);
  switch (d->row) {
    case 128: return launch_latent<4, 2>(st, a);
    case 256: return launch_latent<8, 2>(st, a);
    case 320: return launch_latent<10, 2>(st, a);
    default: return launch_latent<18, 4>(st, a);
  }
}

extern "C" int tnx_gate_mul(void* stream, const tnx_gate_mul_desc* d) {
  TNX_REQUIRE(d && d->M > 0 && d->W > 0 && d->head > 0 && d->W % d->head == 0 && d->y_head >= d->head, "gate_mul: bad shape");
  TNX_REQUIRE(d->y && src_given(d->g) && d->out && d->out_ld >= d->W && d->y_ld >= d->W / d->head * d->y_head, "gate_mul: null pointer or short rows");
  TNX_REQUIRE(known_dtype(d->dtype), "gate_mul: bad dtype %d", d->dtype);
  return d->dtype == TNX_BF16 ? gate_launch<uint16_t>(as_stream(stream), d) : gate_launch<float>(as_stream(stream), d);
}
