// Lightning attention: per head a matrix state S [dim, vdim] in fp32,
//   S_t = decay S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,
// with q, k, v = silu of a fused projection's columns.  o leaves in fp32 [rows, H * vdim]; the state
// [B, H, dim, vdim] is read (from column 0 on: taken as zero) and written back.
//
//   lightning_chunk_kernel   prompts: 64 tokens at a time on MFMAs; a long prompt is cut into spans
//                            that run in parallel, their start states formed by a scan over spans
//   lightning_step_kernel    one token per sequence: one pass over the state
//   lightning_any_kernel     any sizes and fp32: token by token
#include <string.h>

#include <mutex>

#include "decoder.h"

namespace {

struct LightArgs {
  int64_t B, T;
  int H, dk, dv;
  const float* decay;      // [H]
  const int32_t* starts;   // [B]
  const int32_t* col_ptr;
  int64_t k_off, v_off, o_ld;
  float* state;
  float* o;
  // chunk kernel
  const uint16_t* y;
  int64_t y_ld;
  int n_spans, span;       // span: tokens, a multiple of 64
  float* ws;               // [B, H, n_spans, dk, dv]
};

__device__ __forceinline__ float silu_fast(float z) {
  return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
}

template <typename T>
__global__ __launch_bounds__(256) void lightning_any_kernel(const LightArgs a, const RowSrc<T> src) {
  extern __shared__ float sm[];   // q [dk], k [dk]
  const int h = blockIdx.x, tid = threadIdx.x;
  const int64_t b = blockIdx.y;
  const int col0 = *a.col_ptr, start = a.starts[b];
  const float lam = a.decay[h];
  float* S = a.state + (b * a.H + h) * (int64_t)a.dk * a.dv;
  bool fresh = col0 <= start;     // no token of this sequence has run yet
  for (int64_t t = max(0, start - col0); t < a.T; ++t) {
    const int64_t row = b * a.T + t;
    __syncthreads();
    for (int i = tid; i < a.dk; i += 256) {
      sm[i] = silu_f32(src.get(row, (int64_t)h * a.dk + i));
      sm[a.dk + i] = silu_f32(src.get(row, a.k_off + (int64_t)h * a.dk + i));
    }
    __syncthreads();
    for (int d = tid; d < a.dv; d += 256) {
      const float v = silu_f32(src.get(row, a.v_off + (int64_t)h * a.dv + d));
      float acc = 0.f;
#pragma unroll 4
      for (int i = 0; i < a.dk; ++i) {
        const int64_t at = (int64_t)i * a.dv + d;
        const float s = (fresh ? 0.f : lam * S[at]) + sm[a.dk + i] * v;
        S[at] = s;
        acc += sm[i] * s;
      }
      a.o[row * a.o_ld + (int64_t)h * a.dv + d] = acc;
    }
    fresh = false;
  }
  // rows in front of the sequence: defined values for the norms behind
  for (int64_t t = 0; t < min((int64_t)max(0, start - col0), a.T); ++t)
    for (int d = tid; d < a.dv; d += 256) a.o[(b * a.T + t) * a.o_ld + (int64_t)h * a.dv + d] = 0.f;
}

// One token: a thread owns four value columns and every NG-th row of the state.
template <typename T>
__global__ __launch_bounds__(256) void lightning_step_kernel(const LightArgs a, const RowSrc<T> src) {
  extern __shared__ __align__(16) float sm[];   // q [dk], k [dk], then the partial outputs [256][4]
  const int h = blockIdx.x, tid = threadIdx.x;
  const int64_t b = blockIdx.y;
  const int nc = a.dv / 4, ng = 256 / nc, grp = tid / nc, c = tid % nc;
  const bool fresh = *a.col_ptr <= a.starts[b];
  const float lam = fresh ? 0.f : a.decay[h];
  f32x4* part = reinterpret_cast<f32x4*>(sm + (2 * a.dk + 3) / 4 * 4);
  f32x4* S = reinterpret_cast<f32x4*>(a.state + (b * a.H + h) * (int64_t)a.dk * a.dv);
  // the first rows of the state are on their way while q, k and v arrive
  constexpr int PF = 8;
  f32x4 s[PF];
  const bool mine = grp < ng;
#pragma unroll
  for (int u = 0; u < PF; ++u) {
    const int i = grp + u * ng;
    s[u] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (mine && i < a.dk && !fresh) s[u] = __builtin_nontemporal_load(&S[(int64_t)i * nc + c]);
  }
  for (int i = tid; i < a.dk; i += 256) {
    sm[i] = silu_f32(src.get(b, (int64_t)h * a.dk + i));
    sm[a.dk + i] = silu_f32(src.get(b, a.k_off + (int64_t)h * a.dk + i));
  }
  f32x4 v = f32x4{0.f, 0.f, 0.f, 0.f}, acc = v;
  if (mine)
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = silu_f32(src.get(b, a.v_off + (int64_t)h * a.dv + c * 4 + e));
  __syncthreads();
  if (mine)
    for (int i0 = grp; i0 < a.dk; i0 += PF * ng) {
      f32x4 nx[PF];
#pragma unroll
      for (int u = 0; u < PF; ++u) {
        const int i = i0 + (PF + u) * ng;
        nx[u] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (i < a.dk && !fresh) nx[u] = __builtin_nontemporal_load(&S[(int64_t)i * nc + c]);
      }
#pragma unroll
      for (int u = 0; u < PF; ++u) {
        const int i = i0 + u * ng;
        if (i < a.dk) {
          const f32x4 w = lam * s[u] + sm[a.dk + i] * v;
          __builtin_nontemporal_store(w, &S[(int64_t)i * nc + c]);
          acc += sm[i] * w;
        }
        s[u] = nx[u];
      }
    }
  part[tid] = acc;
  __syncthreads();
  if (tid < nc) {
    f32x4 t = part[tid];
    for (int gq = 1; gq < ng; ++gq) t += part[gq * nc + tid];
    float* o = a.o + b * a.o_ld + (int64_t)h * a.dv + tid * 4;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = t[e];
  }
}

constexpr int kChunk = 64, kTLD = kChunk + 8;
constexpr size_t light_smem_bytes(int kt) {
  // Q, K [64][dk + 8]; decayed K^T high and low [dk][72]; V^T [128][72] (bf16); two power tables
  return (size_t)(2 * kChunk * (kt * 32 + 8) + 2 * kt * 32 * kTLD + 128 * kTLD) * 2 + 2 * 80 * 4;
}

// A work-group takes one span of one (row, head) and up to 128 value columns; wave w keeps the state's
// columns 32 w .. + 31 in its accumulators (fp32).  Per chunk of 64 tokens:
//   o = decay^(i+1) (q S) + ((q k^T) . decay^(i-j), j <= i) v
//   S = decay^n S + sum_j decay^(n-1-j) k_j v_j^T
// The accumulator layout of S is, in a permuted order of the head dimension that q's fragments
// follow, the B operand of q S; likewise the scores (computed transposed) are the A operand of the
// product with v.  fp32 operands (S, decayed k, weighted scores) enter as a high and a low bf16 part.
// STATES: only the span's own contribution to the state is formed (into ws).
template <int KT, bool STATES>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, 1))) void lightning_chunk_kernel(const LightArgs a) {
  constexpr int DK = KT * 32, QLD = DK + 8;
  extern __shared__ __align__(16) unsigned char smem[];
  uint16_t* qs = reinterpret_cast<uint16_t*>(smem);
  uint16_t* ks = qs + kChunk * QLD;
  uint16_t* kth = ks + kChunk * QLD;
  uint16_t* ktl = kth + DK * kTLD;
  uint16_t* vt = ktl + DK * kTLD;
  float* pw = reinterpret_cast<float*>(vt + 128 * kTLD);   // decay^i, i = 0..64
  float* pw1 = pw + 80;                                    // decay^(i+1), i = 0..63
  const int tid = threadIdx.x, lane = tid & 63, l32 = lane & 31, lh = lane >> 5;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int span = blockIdx.x % a.n_spans, slice = blockIdx.x / a.n_spans;
  const int h = blockIdx.y;
  const int64_t b = blockIdx.z;
  if (STATES && span == a.n_spans - 1) return;             // nothing starts from the last span's state
  const int col0 = *a.col_ptr, start = a.starts[b];
  const float lam = a.decay[h];
  if (tid <= kChunk) {
    pw[tid] = powf(lam, (float)tid);
    if (tid < kChunk) pw1[tid] = powf(lam, (float)(tid + 1));
  }
  const int dv0 = slice * 128, dvw = dv0 + wave * 32;      // this wave's first value column
  const bool active = dvw < a.dv;
  const int t_begin = span * a.span, t_end = min((int)a.T, t_begin + a.span);
  const int dcol = dvw + l32;                              // this lane's value column
  const bool dok = dcol < a.dv;

  f32x16 S[KT];
  {
    const float* init = nullptr;
    if (!STATES) {
      if (a.n_spans > 1) init = a.ws + ((b * a.H + h) * a.n_spans + span) * (int64_t)a.dk * a.dv;
      else if (col0 > start) init = a.state + (b * a.H + h) * (int64_t)a.dk * a.dv;
    }
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int r = kt * 32 + 8 * (i >> 2) + 4 * lh + (i & 3);
        S[kt][i] = init && dok && r < a.dk ? init[(int64_t)r * a.dv + dcol] : 0.f;
      }
  }

  // staging: item = (pair of tokens, eight dimensions)
  constexpr int QI = 32 * (DK / 8) / 256 > 0 ? 32 * (DK / 8) / 256 : 1;   // items per thread of q and of k
  constexpr int VI = 2;                                                   // 32 pairs x 16 chunks of v
  u32x4 qr[QI][2], kr[QI][2], vr[VI][2];
  const u32x4 zero = u32x4{0, 0, 0, 0};
  auto fetch = [&](int t0) {
#pragma unroll
    for (int c = 0; c < QI; ++c) {
      const int it = c * 256 + tid, pr = it / (DK / 8), ch = it % (DK / 8);
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int t = t0 + 2 * pr + e;
        const bool ok = pr < 32 && ch * 8 < a.dk && t < t_end && col0 + t >= start;
        const uint16_t* p = a.y + (b * a.T + t) * a.y_ld + (int64_t)h * a.dk + ch * 8;
        if (!STATES) qr[c][e] = ok ? *reinterpret_cast<const u32x4*>(p) : zero;
        kr[c][e] = ok ? *reinterpret_cast<const u32x4*>(p + a.k_off) : zero;
      }
    }
#pragma unroll
    for (int c = 0; c < VI; ++c) {
      const int it = c * 256 + tid, pr = it / 16, d = dv0 + (it % 16) * 8;
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int t = t0 + 2 * pr + e;
        const bool ok = d < a.dv && t < t_end && col0 + t >= start;
        vr[c][e] = ok ? *reinterpret_cast<const u32x4*>(a.y + (b * a.T + t) * a.y_ld + a.v_off + (int64_t)h * a.dv + d) : zero;
      }
    }
  };
  auto act8 = [&](const u32x4& v, float (&f)[8]) {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      f[2 * j] = silu_fast(bflo(v[j]));
      f[2 * j + 1] = silu_fast(bfhi(v[j]));
    }
  };

  // chunks wholly in front of the sequence change nothing
  int t0 = t_begin;
  if (start > col0) t0 = max(t_begin, t_begin + (start - col0 - t_begin) / kChunk * kChunk);
  if (!STATES && active && dok)
    for (int t = t_begin + lh; t < min(t0, t_end); t += 2) a.o[(b * a.T + t) * a.o_ld + (int64_t)h * a.dv + dcol] = 0.f;
  if (t0 < t_end) fetch(t0);
  for (; t0 < t_end; t0 += kChunk) {
    const int n = min(kChunk, t_end - t0);
    __syncthreads();    // the readers of the chunk before are done (first turn: the tables are written)
#pragma unroll
    for (int c = 0; c < QI; ++c) {
      const int it = c * 256 + tid, pr = it / (DK / 8), ch = it % (DK / 8);
      if (pr >= 32) continue;
      float f0[8], f1[8];
      if (!STATES) {
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          act8(qr[c][e], f0);
          *reinterpret_cast<u32x4*>(&qs[(2 * pr + e) * QLD + ch * 8]) =
              u32x4{cvt_pk_bf16(f0[0], f0[1]), cvt_pk_bf16(f0[2], f0[3]), cvt_pk_bf16(f0[4], f0[5]), cvt_pk_bf16(f0[6], f0[7])};
        }
      }
      act8(kr[c][0], f0);
      act8(kr[c][1], f1);
      const u32x4 k0 = {cvt_pk_bf16(f0[0], f0[1]), cvt_pk_bf16(f0[2], f0[3]), cvt_pk_bf16(f0[4], f0[5]), cvt_pk_bf16(f0[6], f0[7])};
      const u32x4 k1 = {cvt_pk_bf16(f1[0], f1[1]), cvt_pk_bf16(f1[2], f1[3]), cvt_pk_bf16(f1[4], f1[5]), cvt_pk_bf16(f1[6], f1[7])};
      if (!STATES) {
        *reinterpret_cast<u32x4*>(&ks[(2 * pr) * QLD + ch * 8]) = k0;
        *reinterpret_cast<u32x4*>(&ks[(2 * pr + 1) * QLD + ch * 8]) = k1;
      }
      // (tokens past n hold zeros: any power will do)
      const float d0 = pw[max(n - 1 - 2 * pr, 0)], d1 = pw[max(n - 2 - 2 * pr, 0)];
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float x0 = (j & 1) ? bfhi(k0[j >> 1]) : bflo(k0[j >> 1]), x1 = (j & 1) ? bfhi(k1[j >> 1]) : bflo(k1[j >> 1]);
        uint32_t hi, lo;
        split2(x0 * d0, x1 * d1, hi, lo);
        *reinterpret_cast<uint32_t*>(&kth[(ch * 8 + j) * kTLD + 2 * pr]) = hi;
        *reinterpret_cast<uint32_t*>(&ktl[(ch * 8 + j) * kTLD + 2 * pr]) = lo;
      }
    }
#pragma unroll
    for (int c = 0; c < VI; ++c) {
      const int it = c * 256 + tid, pr = it / 16, ch = it % 16;
      float f0[8], f1[8];
      act8(vr[c][0], f0);
      act8(vr[c][1], f1);
#pragma unroll
      for (int j = 0; j < 8; ++j) *reinterpret_cast<uint32_t*>(&vt[(ch * 8 + j) * kTLD + 2 * pr]) = cvt_pk_bf16(f0[j], f1[j]);
    }
    __syncthreads();
    if (t0 + kChunk < t_end) fetch(t0 + kChunk);
    if (!active) continue;                                 // (wave-uniform)
    if constexpr (!STATES) {
      f32x16 O[2];
#pragma unroll
      for (int qt = 0; qt < 2; ++qt)
#pragma unroll
        for (int i = 0; i < 16; ++i) O[qt][i] = 0.f;
      // q S: k index 8 lh + 4 b + e of step s <-> head dimension 32 kt + 16 s + 8 b + 4 lh + e
#pragma unroll
      for (int kt = 0; kt < KT; ++kt)
#pragma unroll
        for (int s = 0; s < 2; ++s) {
          u32x4 bh, bl;
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            uint32_t hi, lo;
            split2(S[kt][8 * s + 2 * r], S[kt][8 * s + 2 * r + 1], hi, lo);
            bh[r] = hi;
            bl[r] = lo;
          }
#pragma unroll
          for (int qt = 0; qt < 2; ++qt) {
            const uint16_t* p = &qs[(qt * 32 + l32) * QLD + kt * 32 + 16 * s + 4 * lh];
            const u32x2 p0 = *reinterpret_cast<const u32x2*>(p), p1 = *reinterpret_cast<const u32x2*>(p + 8);
            const u32x4 af = {p0[0], p0[1], p1[0], p1[1]};
            O[qt] = mfma32(af, bh, O[qt]);
            O[qt] = mfma32(af, bl, O[qt]);
          }
        }
#pragma unroll
      for (int qt = 0; qt < 2; ++qt)
#pragma unroll
        for (int bb = 0; bb < 4; ++bb) {
          const f32x4 w = *reinterpret_cast<const f32x4*>(&pw1[qt * 32 + 8 * bb + 4 * lh]);
#pragma unroll
          for (int e = 0; e < 4; ++e) O[qt][4 * bb + e] *= w[e];
        }
      // inside the chunk
#pragma unroll
      for (int qt = 0; qt < 2; ++qt)
#pragma unroll
        for (int jt = 0; jt <= qt; ++jt) {
          f32x16 st;
#pragma unroll
          for (int i = 0; i < 16; ++i) st[i] = 0.f;
#pragma unroll
          for (int s = 0; s < 2 * KT; ++s)
            st = mfma32(*reinterpret_cast<const u32x4*>(&ks[(jt * 32 + l32) * QLD + 16 * s + 8 * lh]),
                        *reinterpret_cast<const u32x4*>(&qs[(qt * 32 + l32) * QLD + 16 * s + 8 * lh]), st);
          // lane: query qt * 32 + l32; register 4 b + e: key jt * 32 + 8 b + 4 lh + e
#pragma unroll
          for (int i = 0; i < 16; ++i) {
            const int d = (qt - jt) * 32 + l32 - (8 * (i >> 2) + 4 * lh + (i & 3));
            const float w = pw[max(d, 0)];
            st[i] = d >= 0 ? st[i] * w : 0.f;
          }
#pragma unroll
          for (int s = 0; s < 2; ++s) {
            u32x4 ah, al;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              uint32_t hi, lo;
              split2(st[8 * s + 2 * r], st[8 * s + 2 * r + 1], hi, lo);
              ah[r] = hi;
              al[r] = lo;
            }
            const uint16_t* p = &vt[(wave * 32 + l32) * kTLD + jt * 32 + 16 * s + 4 * lh];
            const u32x2 p0 = *reinterpret_cast<const u32x2*>(p), p1 = *reinterpret_cast<const u32x2*>(p + 8);
            const u32x4 bf = {p0[0], p0[1], p1[0], p1[1]};
            O[qt] = mfma32(ah, bf, O[qt]);
            O[qt] = mfma32(al, bf, O[qt]);
          }
        }
      if (dok)
#pragma unroll
        for (int qt = 0; qt < 2; ++qt)
#pragma unroll
          for (int i = 0; i < 16; ++i) {
            const int r = qt * 32 + 8 * (i >> 2) + 4 * lh + (i & 3);
            if (r < n) a.o[(b * a.T + t0 + r) * a.o_ld + (int64_t)h * a.dv + dcol] = O[qt][i];
          }
    }
    // the state behind this chunk
    const float dn = pw[n];
    u32x4 bv[4];
#pragma unroll
    for (int s = 0; s < 4; ++s) bv[s] = *reinterpret_cast<const u32x4*>(&vt[(wave * 32 + l32) * kTLD + 16 * s + 8 * lh]);
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
#pragma unroll
      for (int i = 0; i < 16; ++i) S[kt][i] *= dn;
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        S[kt] = mfma32(*reinterpret_cast<const u32x4*>(&kth[(kt * 32 + l32) * kTLD + 16 * s + 8 * lh]), bv[s], S[kt]);
        S[kt] = mfma32(*reinterpret_cast<const u32x4*>(&ktl[(kt * 32 + l32) * kTLD + 16 * s + 8 * lh]), bv[s], S[kt]);
      }
    }
  }
  if (!active || !dok) return;
  float* dst = nullptr;
  if (STATES) dst = a.ws + ((b * a.H + h) * a.n_spans + span) * (int64_t)a.dk * a.dv;
  else if (span == a.n_spans - 1) dst = a.state + (b * a.H + h) * (int64_t)a.dk * a.dv;
  if (dst)
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int r = kt * 32 + 8 * (i >> 2) + 4 * lh + (i & 3);
        if (r < a.dk) dst[(int64_t)r * a.dv + dcol] = S[kt][i];
      }
}

// the spans' own contributions -> the state each span starts from, in place
__global__ __launch_bounds__(256) void lightning_scan_kernel(const LightArgs a) {
  const int64_t n = (int64_t)a.dk * a.dv, i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  const int h = blockIdx.y;
  const int64_t b = blockIdx.z;
  if (i >= n) return;
  const float ls = powf(a.decay[h], (float)a.span);
  float cur = *a.col_ptr > a.starts[b] ? a.state[(b * a.H + h) * n + i] : 0.f;
  float* p = a.ws + (b * a.H + h) * a.n_spans * n + i;
  for (int s = 0; s < a.n_spans; ++s) {
    const float u = s + 1 < a.n_spans ? p[s * n] : 0.f;
    p[s * n] = cur;
    cur = ls * cur + u;
  }
}

template <int KT>
int launch_chunk(hipStream_t st, const LightArgs& a) {
  static std::once_flag once;
  static hipError_t e = hipSuccess;
  constexpr size_t kSmem = light_smem_bytes(KT);
  std::call_once(once, [] {
    e = hipFuncSetAttribute(reinterpret_cast<const void*>(&lightning_chunk_kernel<KT, false>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kSmem);
    if (e == hipSuccess)
      e = hipFuncSetAttribute(reinterpret_cast<const void*>(&lightning_chunk_kernel<KT, true>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kSmem);
  });
  if (e != hipSuccess) {
    tnx_set_error("lightning: cannot raise the dynamic LDS limit: %s", hipGetErrorString(e));
    return TNX_ELAUNCH;
  }
  const dim3 grid((unsigned)(a.n_spans * cdiv(a.dv, 128)), (unsigned)a.H, (unsigned)a.B);
  if (a.n_spans > 1) {
    hipLaunchKernelGGL((lightning_chunk_kernel<KT, true>), grid, dim3(256), kSmem, st, a);
    hipLaunchKernelGGL(lightning_scan_kernel, dim3((unsigned)cdiv((int64_t)a.dk * a.dv, 256), (unsigned)a.H, (unsigned)a.B), dim3(256), 0, st, a);
  }
  hipLaunchKernelGGL((lightning_chunk_kernel<KT, false>), grid, dim3(256), kSmem, st, a);
  TNX_CHECK_LAUNCH("lightning_chunk");
  return TNX_OK;
}

// work-groups of a prompt pass that fill the device; shorter spans cost state traffic
int span_tokens(int64_t B, int64_t T, int H) {
  const int64_t per = B * H;
  int64_t spans = per >= 256 ? 1 : cdiv(512, per);
  int64_t span = cdiv(cdiv(T, spans), kChunk) * kChunk;
  if (span < 2 * kChunk) span = 2 * kChunk;
  return (int)span;
}

}  // namespace

extern "C" size_t tnx_lightning_ws_bytes(int64_t B, int64_t T, int H, int dk, int dv) {
  if (T <= 1 || B <= 0) return 0;
  const int64_t spans = cdiv(T, span_tokens(B, T, H));
  return spans > 1 ? (size_t)(B * H * spans) * (size_t)dk * (size_t)dv * 4 : 0;
}

extern "C" int tnx_lightning(void* stream, const tnx_lightning_desc* d) {
  TNX_REQUIRE(d, "lightning: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->T > 0 && d->H > 0 && d->dk > 0 && d->dv > 0, "lightning: bad shape");
  TNX_REQUIRE(d->decay && d->starts && d->col_ptr && d->state && d->o && src_given(d->y), "lightning: null pointer");
  TNX_REQUIRE(d->o_ld >= (int64_t)d->H * d->dv && d->dk <= 8192, "lightning: short output rows or a head size above 8192");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "lightning: bad dtype %d", d->dtype);
  TNX_REQUIRE(d->B <= 65535 && d->H <= 65535, "lightning: too many rows or heads");
  LightArgs a;
  memset(&a, 0, sizeof(a));
  a.B = d->B; a.T = d->T; a.H = d->H; a.dk = d->dk; a.dv = d->dv; a.decay = d->decay; a.starts = d->starts;
  a.col_ptr = d->col_ptr; a.k_off = d->k_off; a.v_off = d->v_off; a.o_ld = d->o_ld; a.state = d->state; a.o = d->o;
  hipStream_t st = as_stream(stream);
  const bool bf = d->dtype == TNX_BF16;
  const RowSrc<uint16_t> s16{(const uint16_t*)d->y.y, d->y.ws, d->y.split_k, d->y.plane, d->y.ld};
  const RowSrc<float> s32{(const float*)d->y.y, d->y.ws, d->y.split_k, d->y.plane, d->y.ld};
  const dim3 per((unsigned)d->H, (unsigned)d->B);
  if (d->T == 1 && d->dv % 4 == 0 && d->dv <= 1024 && d->dk <= 4096) {
    const size_t lds = (size_t)((2 * d->dk + 3) / 4 * 4 + 1024) * 4;
    if (bf) hipLaunchKernelGGL(lightning_step_kernel<uint16_t>, per, dim3(256), lds, st, a, s16);
    else hipLaunchKernelGGL(lightning_step_kernel<float>, per, dim3(256), lds, st, a, s32);
    TNX_CHECK_LAUNCH("lightning_step");
    return TNX_OK;
  }
  if (bf && d->T > 1 && d->y.split_k <= 1 && d->dk % 8 == 0 && d->dk <= 256 && d->dv % 8 == 0 && d->k_off % 8 == 0 && d->v_off % 8 == 0 &&
      d->y.ld % 8 == 0 && d->T < (1 << 30)) {
    a.y = (const uint16_t*)d->y.y; a.y_ld = d->y.ld;
    a.span = span_tokens(d->B, d->T, d->H);
    a.n_spans = (int)cdiv(d->T, a.span);
    a.ws = d->ws;
    TNX_REQUIRE(a.n_spans == 1 || d->ws, "lightning: a long prompt needs the workspace of tnx_lightning_ws_bytes");
    if (d->dk <= 32) return launch_chunk<1>(st, a);
    if (d->dk <= 64) return launch_chunk<2>(st, a);
    if (d->dk <= 128) return launch_chunk<4>(st, a);
    return launch_chunk<8>(st, a);
  }
  const size_t lds = (size_t)2 * d->dk * 4;
  if (bf) hipLaunchKernelGGL(lightning_any_kernel<uint16_t>, per, dim3(256), lds, st, a, s16);
  else hipLaunchKernelGGL(lightning_any_kernel<float>, per, dim3(256), lds, st, a, s32);
  TNX_CHECK_LAUNCH("lightning_any");
  return TNX_OK;
}
