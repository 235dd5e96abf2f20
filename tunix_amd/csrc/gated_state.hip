// Linear attention with a forget gate per channel, whose complement writes (HGRN2): per head a matrix state S [dim, vdim]
// in fp32,
//   f = lower + (1 - lower) sigmoid(z + bias),   S_t = diag(f_t) S_(t-1) + (1 - f_t) v_t^T,   o_t = S_t^T silu(q_t).
// o leaves in fp32 [rows, H * vdim]; the state [B, H, dim, vdim] is read (from column 0 on: taken as zero) and written back.
//
//   gated_chunk_kernel   prompts: 32 tokens at a time on MFMAs; a long prompt is cut into spans that run in
//                        parallel, their start states formed by a scan over spans
//   gated_step_kernel    one token per sequence: one pass over the state, optionally the heads' norms behind it
//   gated_any_kernel     any sizes and fp32: token by token
#include <string.h>

#include <mutex>

#include "decoder.h"

namespace {

typedef float f32x2 __attribute__((ext_vector_type(2)));

struct GateArgs {
  int64_t B, T;
  int H, dk, dv;
  const float* bias;       // [H * dk]
  const float* lower;      // [H * dk]
  const int32_t* starts;   // [B]
  const int32_t* col_ptr;
  int64_t q_off, v_off, f_off, o_ld;
  float* state;
  float* o;
  // chunk kernel
  int n_spans, span;       // span: tokens, a multiple of 32
  float* ws;               // states [B, H, n_spans, dk, dv], then decays [B, H, n_spans, dk]
  // step kernel
  const float* norm_w;     // [dv] or null
  float eps;
  void* out;
  int64_t out_ld;
  int out_frag;
};

// f and 1 - f, each to its own relative precision
template <bool FAST>
__device__ __forceinline__ void forget(float z, float lower, float& f, float& k) {
  const float e = FAST ? __builtin_amdgcn_exp2f(-1.4426950408889634f * fabsf(z)) : expf(-fabsf(z));
  const float big = FAST ? __builtin_amdgcn_rcpf(1.0f + e) : 1.0f / (1.0f + e), small = e * big;
  f = lower + (1.0f - lower) * (z >= 0.f ? big : small);
  k = (1.0f - lower) * (z >= 0.f ? small : big);
}
__device__ __forceinline__ float silu_fast(float z) {
  return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
}

template <typename T>
__global__ __launch_bounds__(256) void gated_any_kernel(const GateArgs a, const RowSrc<T> src, const RowSrc<float> fs) {
  extern __shared__ float sm[];   // q [dk], f [dk], k [dk]
  const int h = blockIdx.x, tid = threadIdx.x;
  const int64_t b = blockIdx.y, hk = (int64_t)h * a.dk, hv = (int64_t)h * a.dv;
  const int col0 = *a.col_ptr, start = a.starts[b];
  float* S = a.state + (b * a.H + h) * (int64_t)a.dk * a.dv;
  bool fresh = col0 <= start;     // no token of this sequence has run yet
  for (int64_t t = max(0, start - col0); t < a.T; ++t) {
    const int64_t row = b * a.T + t;
    __syncthreads();
    for (int i = tid; i < a.dk; i += 256) {
      sm[i] = silu_f32(src.get(row, a.q_off + hk + i));
      forget<false>(fs.get(row, a.f_off + hk + i) + a.bias[hk + i], a.lower[hk + i], sm[a.dk + i], sm[2 * a.dk + i]);
    }
    __syncthreads();
    for (int d = tid; d < a.dv; d += 256) {
      const float v = src.get(row, a.v_off + hv + d);
      float acc = 0.f;
#pragma unroll 4
      for (int i = 0; i < a.dk; ++i) {
        const int64_t at = (int64_t)i * a.dv + d;
        const float s = (fresh ? 0.f : sm[a.dk + i] * S[at]) + sm[2 * a.dk + i] * v;
        S[at] = s;
        acc += sm[i] * s;
      }
      a.o[row * a.o_ld + hv + d] = acc;
    }
    fresh = false;
  }
  // rows in front of the sequence: defined values for the norms behind
  for (int64_t t = 0; t < min((int64_t)max(0, start - col0), a.T); ++t)
    for (int d = tid; d < a.dv; d += 256) a.o[(b * a.T + t) * a.o_ld + hv + d] = 0.f;
}

// One token: a thread owns four value columns and every NG-th row of the state.
template <typename TY, typename T>   // types of y's finished rows and of the normed output
__global__ __launch_bounds__(256) void gated_step_kernel(const GateArgs a, const RowSrc<TY> src, const RowSrc<float> fs) {
  extern __shared__ __align__(16) float sm[];   // q, f, k [dk] each, then the partial outputs [256][4]
  __shared__ float red[4];
  const int h = blockIdx.x, tid = threadIdx.x;
  const int64_t b = blockIdx.y, hk = (int64_t)h * a.dk, hv = (int64_t)h * a.dv;
  const int nc = a.dv / 4, ng = 256 / nc, grp = tid / nc, c = tid % nc;
  const bool fresh = *a.col_ptr <= a.starts[b];
  f32x4* part = reinterpret_cast<f32x4*>(sm + (3 * a.dk + 3) / 4 * 4);
  f32x4* S = reinterpret_cast<f32x4*>(a.state + (b * a.H + h) * (int64_t)a.dk * a.dv);
  // the first rows of the state are on their way while q, f and v arrive
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
    sm[i] = silu_f32(src.get(b, a.q_off + hk + i));
    forget<false>(fs.get(b, a.f_off + hk + i) + a.bias[hk + i], a.lower[hk + i], sm[a.dk + i], sm[2 * a.dk + i]);
  }
  f32x4 v = f32x4{0.f, 0.f, 0.f, 0.f}, acc = v;
  if (mine)
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = src.get(b, a.v_off + hv + c * 4 + e);
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
          const f32x4 w = sm[a.dk + i] * s[u] + sm[2 * a.dk + i] * v;
          __builtin_nontemporal_store(w, &S[(int64_t)i * nc + c]);
          acc += sm[i] * w;
        }
        s[u] = nx[u];
      }
    }
  part[tid] = acc;
  __syncthreads();
  f32x4 t = f32x4{0.f, 0.f, 0.f, 0.f};
  if (tid < nc) {
    t = part[tid];
    for (int gq = 1; gq < ng; ++gq) t += part[gq * nc + tid];
  }
  if (!a.norm_w) {   // (uniform)
    if (tid < nc) *reinterpret_cast<f32x4*>(a.o + b * a.o_ld + hv + tid * 4) = t;
    return;
  }
  const float ss = wave_sum(t[0] * t[0] + t[1] * t[1] + t[2] * t[2] + t[3] * t[3]);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  if (tid >= nc) return;
  const float r = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.dv + a.eps);
  T* out = reinterpret_cast<T*>(a.out);
  const int64_t col = hv + tid * 4, at = a.out_frag ? frag_index(b, col, a.out_ld) : b * a.out_ld + col;   // (runs of eight stay together)
#pragma unroll
  for (int e = 0; e < 4; ++e) st_elem(out, at + e, t[e] * r * a.norm_w[tid * 4 + e]);
}

// ---- prompts ------------------------------------------------------------------------------------
// Two values of a row, with a k split's planes summed.
template <typename T>
__device__ __forceinline__ f32x2 get2(const RowSrc<T>& s, int64_t row, int64_t col) {
  const int64_t o = row * s.ld + col;
  f32x2 v = f32x2{0.f, 0.f};
  if (s.split > 1) {
    for (int z = 0; z < s.split; ++z) v += *reinterpret_cast<const f32x2*>(s.ws + z * s.plane + o);
  } else if constexpr (sizeof(T) == 2) {
    const uint32_t u = *reinterpret_cast<const uint32_t*>(s.y + o);
    v = f32x2{bflo(u), bfhi(u)};
  } else {
    v = *reinterpret_cast<const f32x2*>(s.y + o);
  }
  return v;
}

constexpr int kTok = 32, kTokLd = kTok + 8;
// LDS of the chunk kernel, in bytes from the start
template <int DK>
struct GateLds {
  static constexpr int LD = DK + 8;                       // row of an operand, bf16
  static constexpr int set = 3 * 16 * LD * 2;             // q [16], k high [16], k low [16]
  static constexpr int qhat = 3 * set;                    // [32][LD], behind the three sets of the second phase
  static constexpr int kt = qhat + kTok * LD * 2;         // high and low [DK][kTokLd]
  static constexpr int first = 4 * set, second = kt + 2 * DK * kTokLd * 2;
  static constexpr int vt = first > second ? first : second;   // [128][kTokLd]
  static constexpr int score = vt + 128 * kTokLd * 2;     // high and low [32][kTokLd]
  static constexpr int total = score + 2 * kTok * kTokLd * 2;   // fp32: per token group [512 / DK][DK], then of the chunk [DK]
  static constexpr int bytes = total + (512 + DK) * 4;
  static constexpr int states_total = (2 * DK + 128) * kTokLd * 2, states_bytes = states_total + (512 + DK) * 4;   // k^T, v^T, totals alone
};

// A work-group takes one span of one (row, head) and up to 128 value columns; wave w keeps the state's columns
// 32 w .. + 31 in its accumulators (fp32).  Per chunk of 32 tokens:
//   o = (q . D(i)) S + A v,   A_ij = sum_d q_i k_j prod_(j < s <= i) f_s  (j <= i),   S = D S + sum_j (k_j . R(j)) v_j^T
// with D(i) the product of f up to token i, R(j) the product behind token j.  A decay of its own per channel does not
// divide out of a chunk without overflow, so A is put together from levels s = 16, 8, 4, 2, 1: for a pair of neighbouring
// blocks of s tokens, j in the first and i in the second, the product splits at the border between the blocks into one over
// the second block up to i, which scales q_i, and one over the first block behind j, which scales k_j -- both at most 1.  Every
// token has one part per level, so a level is one 16 x 16 product; the diagonal (q_i . k_i) is two more, odd tokens and
// even ones.  The scales need no logarithm: a level's products are the level's before times a block's total.
// k = 1 - f, the state and A enter the products as a high and a low bf16 part, scaled queries and values as bf16.
// Thread (group, pair) owns DK / 16 neighbouring tokens of two channels.
// STATES: only the span's own contribution to the state and its decays are formed (into ws).
template <int KT, bool STATES, typename TY>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(KT <= 2 || (STATES && KT <= 4) ? 2 : 1, KT <= 2 || STATES ? 2 : 1))) void gated_chunk_kernel(const GateArgs a, const RowSrc<TY> src, const RowSrc<float> fs) {
  constexpr int DK = KT * 32, LD = GateLds<DK>::LD, PAIRS = DK / 2, NG = 256 / PAIRS, TG = kTok / NG;
  static_assert(TG >= 2 && TG <= 16, "tokens of a thread");
  typedef GateLds<DK> Lds;
  extern __shared__ __align__(16) uint8_t smem[];
  uint16_t* kth = reinterpret_cast<uint16_t*>(smem + (STATES ? 0 : Lds::kt));
  uint16_t* ktl = kth + DK * kTokLd;
  uint16_t* vt = reinterpret_cast<uint16_t*>(smem + (STATES ? 2 * DK * kTokLd * 2 : Lds::vt));
  uint16_t* sch = reinterpret_cast<uint16_t*>(smem + Lds::score);
  uint16_t* scl = sch + kTok * kTokLd;
  float* tot = reinterpret_cast<float*>(smem + (STATES ? Lds::states_total : Lds::total));
  float* all = tot + 512;
  const int tid = threadIdx.x, lane = tid & 63, l32 = lane & 31, lh = lane >> 5, l16 = lane & 15, lq = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int pair = tid % PAIRS, grp = tid / PAIRS, ch = pair * 2;
  const int span = blockIdx.x % a.n_spans, slice = blockIdx.x / a.n_spans;
  const int h = blockIdx.y;
  const int64_t b = blockIdx.z, bh = b * a.H + h, hk = (int64_t)h * a.dk, hv = (int64_t)h * a.dv;
  if (STATES && span == a.n_spans - 1) return;             // nothing starts from the last span's state
  const int col0 = *a.col_ptr, start = a.starts[b];
  const int dv0 = slice * 128, dcol = dv0 + wave * 32 + l32;   // this lane's value column
  const bool active = dv0 + wave * 32 < a.dv, dok = dcol < a.dv;
  const int t_begin = span * a.span, t_end = min((int)a.T, t_begin + a.span);
  const bool ch_ok = ch < a.dk;
  f32x2 bias = f32x2{0.f, 0.f}, lower = f32x2{1.f, 1.f};
  if (ch_ok) {
    bias = *reinterpret_cast<const f32x2*>(a.bias + hk + ch);
    lower = *reinterpret_cast<const f32x2*>(a.lower + hk + ch);
  }

  f32x16 S[KT];
  {
    const float* init = nullptr;
    if (!STATES) {
      if (a.n_spans > 1) init = a.ws + (bh * a.n_spans + span) * (int64_t)a.dk * a.dv;
      else if (col0 > start) init = a.state + bh * (int64_t)a.dk * a.dv;
    }
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int r = kt * 32 + 8 * (i >> 2) + 4 * lh + (i & 3);
        S[kt][i] = init && dok && r < a.dk ? init[(int64_t)r * a.dv + dcol] : 0.f;
      }
  }
  if (!STATES) {   // scores above the diagonal stay zero
    for (int i = tid; i < kTok * kTokLd; i += 256) {
      sch[i] = 0;
      scl[i] = 0;
    }
  }
  f32x2 decay = f32x2{1.f, 1.f};   // of the span so far (STATES)

  // the next chunk's rows, as they come (a conversion would wait for the loads)
  constexpr bool RAW = sizeof(TY) == 2;
  f32x2 qr[RAW ? 1 : TG], zr[TG];
  uint32_t qw[RAW ? TG : 1];
  u32x4 vw[2];
  float v0[8], v1[8];
  const int vp = tid >> 4, vd = dv0 + (tid & 15) * 8;      // this thread's pair of tokens and eight value columns
  auto live = [&](int t) { return t < t_end && col0 + t >= start; };
  const int chc = ch_ok ? ch : 0, vdc = vd < a.dv ? vd : 0;
  const TY* yb = src.y + b * a.T * src.ld;
  const float* fb = fs.y + b * a.T * fs.ld + a.f_off + hk + chc;
  auto fetch = [&](int t0) {
    if constexpr (RAW) {   // finished rows: loads of tokens that are not there go to the last one, and are dropped later
#pragma unroll
      for (int u = 0; u < TG; ++u) {
        const int t = min(t0 + grp * TG + u, (int)a.T - 1);
        if constexpr (!STATES) qw[u] = *reinterpret_cast<const uint32_t*>(yb + t * (int)src.ld + a.q_off + hk + chc);
        zr[u] = *reinterpret_cast<const f32x2*>(fb + t * (int)fs.ld);
      }
      const TY* vb = yb + a.v_off + hv + vdc;
#pragma unroll
      for (int e = 0; e < 2; ++e) vw[e] = *reinterpret_cast<const u32x4*>(vb + min(t0 + 2 * vp + e, (int)a.T - 1) * (int)src.ld);
    } else {
#pragma unroll
      for (int u = 0; u < TG; ++u) {
        const int t = t0 + grp * TG + u;
        qr[u] = zr[u] = f32x2{0.f, 0.f};
        if (ch_ok && live(t)) {
          if (!STATES) qr[u] = get2(src, b * a.T + t, a.q_off + hk + ch);
          zr[u] = get2(fs, b * a.T + t, a.f_off + hk + ch);
        }
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) v0[j] = v1[j] = 0.f;
      if (vd < a.dv) {
        if (live(t0 + 2 * vp)) get8(src, b * a.T + t0 + 2 * vp, a.v_off + hv + vd, v0);
        if (live(t0 + 2 * vp + 1)) get8(src, b * a.T + t0 + 2 * vp + 1, a.v_off + hv + vd, v1);
      }
    }
  };
  // a level's operands.  Row of token i in the set: i / 2s * s + i % s, for s below a thread's tokens grp * TG / 2 and a
  // number that depends on the place in the thread alone
  uint8_t* const row0 = smem + (grp * (TG / 2) * LD + ch) * 2;
  auto put_q = [&](uint8_t* at, f32x2 v) { *reinterpret_cast<uint32_t*>(at) = cvt_pk_bf16(v[0], v[1]); };
  auto put_k = [&](uint8_t* at, f32x2 v) {
    uint32_t hi, lo;
    split2(v[0], v[1], hi, lo);
    *reinterpret_cast<uint32_t*>(at + 16 * LD * 2) = hi;
    *reinterpret_cast<uint32_t*>(at + 32 * LD * 2) = lo;
  };
  // a set's 16 x 16 product into the scores: blocks of 2^shift tokens, -1: the diagonal of odd tokens, -2: of even ones
  auto score = [&](int set, int shift) {
    f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
    const uint16_t* p = reinterpret_cast<const uint16_t*>(smem + set * Lds::set) + l16 * LD + lq * 8;
#pragma unroll
    for (int s = 0; s < KT; ++s) {
      const u32x4 q = *reinterpret_cast<const u32x4*>(p + s * 32);
      acc = mfma16(q, *reinterpret_cast<const u32x4*>(p + 16 * LD + s * 32), acc);
      acc = mfma16(q, *reinterpret_cast<const u32x4*>(p + 32 * LD + s * 32), acc);
    }
    // lane: key row l16, query rows 4 lq + e
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int qi = 4 * lq + e, kj = l16;
      int i, j;
      bool ok;
      if (shift >= 0) {
        const int s = 1 << shift;
        ok = qi >> shift == kj >> shift;
        i = qi + (qi & -s) + s;
        j = kj + (kj & -s);
      } else {
        ok = qi == kj;
        i = j = 2 * qi + 2 + shift;
      }
      if (!ok) continue;
      uint32_t hi, lo;
      split2(acc[e], 0.f, hi, lo);
      sch[i * kTokLd + j] = (uint16_t)hi;
      scl[i * kTokLd + j] = (uint16_t)lo;
    }
  };

  // chunks wholly in front of the sequence change nothing
  int t0 = t_begin;
  if (start > col0 + t_begin) t0 = t_begin + (start - col0 - t_begin) / kTok * kTok;
  if (!STATES && active && dok)
    for (int t = t_begin + lh; t < min(t0, t_end); t += 2) a.o[(b * a.T + t) * a.o_ld + hv + dcol] = 0.f;
  constexpr bool AHEAD = KT < 8 || STATES;   // (wide heads leave no registers for the next chunk's rows)
  if (AHEAD && t0 < t_end) fetch(t0);
  for (; t0 < t_end; t0 += kTok) {
    const int n = min(kTok, t_end - t0);
    if (!AHEAD) fetch(t0);
    // gates; tokens that are not there keep everything and write nothing
    f32x2 qp[TG], kq[TG], tt[TG];
#pragma unroll
    for (int u = 0; u < TG; ++u) {
      const bool on = ch_ok && live(t0 + grp * TG + u);
#pragma unroll
      for (int c = 0; c < 2; ++c) {
        float f, k;
        forget<true>(zr[u][c] + bias[c], lower[c], f, k);
        tt[u][c] = on ? f : 1.f;
        kq[u][c] = on ? k : 0.f;
        if constexpr (STATES) qp[u][c] = 0.f;
        else if constexpr (RAW) qp[u][c] = on ? silu_fast(c ? bfhi(qw[u]) : bflo(qw[u])) : 0.f;
        else qp[u][c] = on ? silu_fast(qr[u][c]) : 0.f;
      }
    }
    f32x2 mine = tt[0];
#pragma unroll
    for (int u = 1; u < TG; ++u) mine *= tt[u];
    if constexpr (!STATES) {
      // first phase: the diagonal and levels 1 and 2
#pragma unroll
      for (int u = 0; u < TG; ++u) {
        uint8_t* at = row0 + (u & 1 ? 0 : Lds::set) + u / 2 * LD * 2;
        put_q(at, qp[u]);
        put_k(at, kq[u]);
        qp[u] *= tt[u];
      }
    }
    *reinterpret_cast<f32x2*>(tot + grp * DK + ch) = mine;
    // levels up to a thread's own tokens
#pragma unroll
    for (int s = 1; s < TG; s *= 2) {
      if constexpr (!STATES)
        if (s <= 2)
#pragma unroll
          for (int u = 0; u < TG; ++u) {
            uint8_t* at = row0 + (s + 1) * Lds::set + (u / (2 * s) * s + u % s) * LD * 2;
            if ((u / s) & 1) put_q(at, qp[u]);
            else put_k(at, kq[u]);
          }
      if (!STATES && s >= 4) continue;   // (formed behind the barrier)
#pragma unroll
      for (int u = 0; u < TG; ++u) {
        if ((u / s) & 1) qp[u] *= tt[u / (2 * s) * 2];
        else kq[u] *= tt[u / (2 * s) * 2 + 1];
      }
#pragma unroll
      for (int p = 0; p < TG / (2 * s); ++p) tt[p] = tt[2 * p] * tt[2 * p + 1];
    }
    if constexpr (!STATES && TG == 2) {   // level 2 lies across threads: a thread's two tokens are one block
#pragma unroll
      for (int u = 0; u < TG; ++u) {
        uint8_t* at = smem + 3 * Lds::set + ((grp / 2 * 2 + u) * LD + ch) * 2;
        if (grp & 1) put_q(at, qp[u]);
        else put_k(at, kq[u]);
      }
    }
    __syncthreads();
    if constexpr (!STATES) {
      score(wave, wave < 2 ? -1 - wave : wave - 2);
      __syncthreads();   // the first phase's operands are read
      // second phase: levels 4, 8 and 16
#pragma unroll
      for (int s = 4; s < TG; s *= 2) {
#pragma unroll
        for (int u = 0; u < TG; ++u) {
          uint8_t* at = row0 + s / 8 * Lds::set + (u / (2 * s) * s + u % s) * LD * 2;
          if ((u / s) & 1) put_q(at, qp[u]);
          else put_k(at, kq[u]);
        }
#pragma unroll
        for (int u = 0; u < TG; ++u) {
          if ((u / s) & 1) qp[u] *= tt[u / (2 * s) * 2];
          else kq[u] *= tt[u / (2 * s) * 2 + 1];
        }
#pragma unroll
        for (int p = 0; p < TG / (2 * s); ++p) tt[p] = tt[2 * p] * tt[2 * p + 1];
      }
    }
    // levels across threads: a thread's tokens lie in one block, whose partner's total comes from the groups' totals
#pragma unroll
    for (int s = TG; s < kTok; s *= 2) {
      const int blk = grp * TG / s, per = s / TG;
      const bool second = blk & 1;
      if constexpr (!STATES)
        if (s >= 4) {
          uint8_t* at = smem + s / 8 * Lds::set + ((blk / 2 * s + grp % per * TG) * LD + ch) * 2;
          if (second)
#pragma unroll
            for (int u = 0; u < TG; ++u) put_q(at + u * LD * 2, qp[u]);
          else
#pragma unroll
            for (int u = 0; u < TG; ++u) put_k(at + u * LD * 2, kq[u]);
        }
      f32x2 other = *reinterpret_cast<const f32x2*>(tot + (blk ^ 1) * per * DK + ch);
#pragma unroll
      for (int g = 1; g < per; ++g) other *= *reinterpret_cast<const f32x2*>(tot + ((blk ^ 1) * per + g) * DK + ch);
      mine *= other;
#pragma unroll
      for (int u = 0; u < TG; ++u) {
        if (second) qp[u] *= other;
        else kq[u] *= other;
      }
    }
    if (grp == 0) *reinterpret_cast<f32x2*>(all + ch) = mine;
    decay *= mine;
#pragma unroll
    for (int u = 0; u < TG; u += 2) {
      if constexpr (!STATES)
#pragma unroll
        for (int e = 0; e < 2; ++e)
          *reinterpret_cast<uint32_t*>(smem + Lds::qhat + ((grp * TG + u + e) * LD + ch) * 2) = cvt_pk_bf16(qp[u + e][0], qp[u + e][1]);
#pragma unroll
      for (int c = 0; c < 2; ++c) {
        uint32_t hi, lo;
        split2(kq[u][c], kq[u + 1][c], hi, lo);
        *reinterpret_cast<uint32_t*>(&kth[(ch + c) * kTokLd + grp * TG + u]) = hi;
        *reinterpret_cast<uint32_t*>(&ktl[(ch + c) * kTokLd + grp * TG + u]) = lo;
      }
    }
    if constexpr (RAW)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        v0[2 * j] = bflo(vw[0][j]);
        v0[2 * j + 1] = bfhi(vw[0][j]);
        v1[2 * j] = bflo(vw[1][j]);
        v1[2 * j + 1] = bfhi(vw[1][j]);
      }
#pragma unroll
    for (int j = 0; j < 8; ++j)   // (a row that is not there may hold anything: nought times it must stay nought)
      *reinterpret_cast<uint32_t*>(&vt[((tid & 15) * 8 + j) * kTokLd + 2 * vp]) =
          cvt_pk_bf16(live(t0 + 2 * vp) ? v0[j] : 0.f, live(t0 + 2 * vp + 1) ? v1[j] : 0.f);
    if (AHEAD && t0 + kTok < t_end) fetch(t0 + kTok);
    __syncthreads();
    f32x16 O;
    u32x4 bv[2];
    if (active)
#pragma unroll
      for (int s = 0; s < 2; ++s) bv[s] = *reinterpret_cast<const u32x4*>(&vt[(wave * 32 + l32) * kTokLd + 16 * s + 8 * lh]);
    if constexpr (!STATES) {
      if (wave < 3) score(wave, 2 + wave);
      if (active) {
#pragma unroll
        for (int i = 0; i < 16; ++i) O[i] = 0.f;
        // q S: k index 8 lh + 4 b + e of step s <-> channel 32 kt + 16 s + 8 b + 4 lh + e
#pragma unroll
        for (int kt = 0; kt < KT; ++kt)
#pragma unroll
          for (int s = 0; s < 2; ++s) {
            u32x4 bh2, bl2;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              uint32_t hi, lo;
              split2(S[kt][8 * s + 2 * r], S[kt][8 * s + 2 * r + 1], hi, lo);
              bh2[r] = hi;
              bl2[r] = lo;
            }
            const uint16_t* p = reinterpret_cast<const uint16_t*>(smem + Lds::qhat) + l32 * LD + kt * 32 + 16 * s + 4 * lh;
            const u32x2 p0 = *reinterpret_cast<const u32x2*>(p), p1 = *reinterpret_cast<const u32x2*>(p + 8);
            const u32x4 af = {p0[0], p0[1], p1[0], p1[1]};
            O = mfma32(af, bh2, O);
            O = mfma32(af, bl2, O);
          }
      }
    }
    // the state behind this chunk
    if (active)
#pragma unroll
      for (int kt = 0; kt < KT; ++kt) {
#pragma unroll
        for (int bb = 0; bb < 4; ++bb) {
          const f32x4 w = *reinterpret_cast<const f32x4*>(&all[kt * 32 + 8 * bb + 4 * lh]);
#pragma unroll
          for (int e = 0; e < 4; ++e) S[kt][4 * bb + e] *= w[e];
        }
#pragma unroll
        for (int s = 0; s < 2; ++s) {
          S[kt] = mfma32(*reinterpret_cast<const u32x4*>(&kth[(kt * 32 + l32) * kTokLd + 16 * s + 8 * lh]), bv[s], S[kt]);
          S[kt] = mfma32(*reinterpret_cast<const u32x4*>(&ktl[(kt * 32 + l32) * kTokLd + 16 * s + 8 * lh]), bv[s], S[kt]);
        }
      }
    __syncthreads();   // all scores are there; the operands, totals and k^T are read
    if constexpr (!STATES) {
      if (active) {
#pragma unroll
        for (int s = 0; s < 2; ++s) {
          O = mfma32(*reinterpret_cast<const u32x4*>(&sch[l32 * kTokLd + 16 * s + 8 * lh]), bv[s], O);
          O = mfma32(*reinterpret_cast<const u32x4*>(&scl[l32 * kTokLd + 16 * s + 8 * lh]), bv[s], O);
        }
        if (dok)
#pragma unroll
          for (int i = 0; i < 16; ++i) {
            const int r = 8 * (i >> 2) + 4 * lh + (i & 3);
            if (r < n) a.o[(b * a.T + t0 + r) * a.o_ld + hv + dcol] = O[i];
          }
      }
    }
  }
  if (STATES && slice == 0 && grp == 0 && ch_ok)
    *reinterpret_cast<f32x2*>(a.ws + a.B * a.H * a.n_spans * (int64_t)a.dk * a.dv + (bh * a.n_spans + span) * a.dk + ch) = decay;
  if (!active || !dok) return;
  float* dst = nullptr;
  if (STATES) dst = a.ws + (bh * a.n_spans + span) * (int64_t)a.dk * a.dv;
  else if (span == a.n_spans - 1) dst = a.state + bh * (int64_t)a.dk * a.dv;
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
__global__ __launch_bounds__(256) void gated_scan_kernel(const GateArgs a) {
  const int64_t n = (int64_t)a.dk * a.dv, i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  const int h = blockIdx.y;
  const int64_t b = blockIdx.z, bh = b * a.H + h;
  if (i >= n) return;
  float cur = *a.col_ptr > a.starts[b] ? a.state[bh * n + i] : 0.f;
  float* p = a.ws + bh * a.n_spans * n + i;
  const float* decay = a.ws + a.B * a.H * a.n_spans * n + bh * a.n_spans * a.dk + i / a.dv;
  for (int s = 0; s < a.n_spans; ++s) {
    const bool more = s + 1 < a.n_spans;
    const float u = more ? p[s * n] : 0.f, f = more ? decay[(int64_t)s * a.dk] : 0.f;
    p[s * n] = cur;
    cur = f * cur + u;
  }
}

template <int KT, typename TY>
int launch_chunk(hipStream_t st, const GateArgs& a, const RowSrc<TY>& src, const RowSrc<float>& fs) {
  static std::once_flag once;
  static hipError_t e = hipSuccess;
  constexpr size_t kSmem = GateLds<KT * 32>::bytes, kStates = GateLds<KT * 32>::states_bytes;
  std::call_once(once, [] {
    e = hipFuncSetAttribute(reinterpret_cast<const void*>(&gated_chunk_kernel<KT, false, TY>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kSmem);
    if (e == hipSuccess)
      e = hipFuncSetAttribute(reinterpret_cast<const void*>(&gated_chunk_kernel<KT, true, TY>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kStates);
  });
  if (e != hipSuccess) {
    tnx_set_error("gated_state: cannot raise the dynamic LDS limit: %s", hipGetErrorString(e));
    return TNX_ELAUNCH;
  }
  const dim3 grid((unsigned)(a.n_spans * cdiv(a.dv, 128)), (unsigned)a.H, (unsigned)a.B);
  if (a.n_spans > 1) {
    hipLaunchKernelGGL((gated_chunk_kernel<KT, true, TY>), grid, dim3(256), kStates, st, a, src, fs);
    hipLaunchKernelGGL(gated_scan_kernel, dim3((unsigned)cdiv((int64_t)a.dk * a.dv, 256), (unsigned)a.H, (unsigned)a.B), dim3(256), 0, st, a);
  }
  hipLaunchKernelGGL((gated_chunk_kernel<KT, false, TY>), grid, dim3(256), kSmem, st, a, src, fs);
  TNX_CHECK_LAUNCH("gated_chunk");
  return TNX_OK;
}
template <typename TY>
int launch_chunk_any(hipStream_t st, const GateArgs& a, const RowSrc<TY>& src, const RowSrc<float>& fs) {
  if (a.dk <= 32) return launch_chunk<1, TY>(st, a, src, fs);
  if (a.dk <= 64) return launch_chunk<2, TY>(st, a, src, fs);
  if (a.dk <= 128) return launch_chunk<4, TY>(st, a, src, fs);
  return launch_chunk<8, TY>(st, a, src, fs);
}

// work-groups of a prompt pass that fill the device; shorter spans cost state traffic
int span_tokens(int64_t B, int64_t T, int H) {
  const int64_t per = B * H;
  const int64_t spans = per >= 256 ? 1 : cdiv(512, per);
  int64_t span = cdiv(cdiv(T, spans), kTok) * kTok;
  if (span < 4 * kTok) span = 4 * kTok;
  return (int)span;
}

}  // namespace

extern "C" int tnx_gated_state_step_ok(int dk, int dv) { return dv % 4 == 0 && dv <= 1024 && dk <= 3072; }

extern "C" size_t tnx_gated_state_ws_bytes(int64_t B, int64_t T, int H, int dk, int dv) {
  if (T <= 1 || B <= 0) return 0;
  const int64_t spans = cdiv(T, span_tokens(B, T, H));
  return spans > 1 ? (size_t)(B * H * spans) * (size_t)dk * (size_t)(dv + 1) * 4 : 0;
}

extern "C" int tnx_gated_state(void* stream, const tnx_gated_state_desc* d) {
  TNX_REQUIRE(d, "gated_state: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->T > 0 && d->H > 0 && d->dk > 0 && d->dv > 0, "gated_state: bad shape");
  TNX_REQUIRE(d->bias && d->lower && d->starts && d->col_ptr && d->state && src_given(d->y) && src_given(d->f), "gated_state: null pointer");
  TNX_REQUIRE(d->q_off >= 0 && d->v_off >= 0 && d->f_off >= 0 && d->q_off + (int64_t)d->H * d->dk <= d->y.ld && d->v_off + (int64_t)d->H * d->dv <= d->y.ld &&
                  d->f_off + (int64_t)d->H * d->dk <= d->f.ld,
              "gated_state: heads outside the rows");
  TNX_REQUIRE(d->dk <= 4096, "gated_state: a head size above 4096");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "gated_state: bad dtype %d", d->dtype);
  TNX_REQUIRE(d->B <= 65535 && d->H <= 65535, "gated_state: too many rows or heads");
  const bool step = d->T == 1 && tnx_gated_state_step_ok(d->dk, d->dv);
  if (d->norm_w) TNX_REQUIRE(step && d->out && d->out_ld >= (int64_t)d->H * d->dv, "gated_state: norms behind the recurrence go with one token and heads the step kernel takes");
  else TNX_REQUIRE(d->o && d->o_ld >= (int64_t)d->H * d->dv, "gated_state: no output rows, or short ones");
  GateArgs a;
  memset(&a, 0, sizeof(a));
  a.B = d->B; a.T = d->T; a.H = d->H; a.dk = d->dk; a.dv = d->dv; a.bias = d->bias; a.lower = d->lower; a.starts = d->starts; a.col_ptr = d->col_ptr;
  a.q_off = d->q_off; a.v_off = d->v_off; a.f_off = d->f_off; a.o_ld = d->o_ld; a.state = d->state; a.o = d->o;
  a.norm_w = d->norm_w; a.eps = d->eps; a.out = d->out; a.out_ld = d->out_ld; a.out_frag = d->out_frag;
  hipStream_t st = as_stream(stream);
  const bool bf = d->dtype == TNX_BF16, y16 = bf && !d->y_f32;
  const int ys = d->y.split_k < 1 ? 1 : d->y.split_k, fsp = d->f.split_k < 1 ? 1 : d->f.split_k;
  const RowSrc<uint16_t> s16{(const uint16_t*)d->y.y, d->y.ws, ys, d->y.plane, d->y.ld};
  const RowSrc<float> s32{(const float*)d->y.y, d->y.ws, ys, d->y.plane, d->y.ld};
  const RowSrc<float> fs{(const float*)d->f.y, d->f.ws, fsp, d->f.plane, d->f.ld};
  const dim3 per((unsigned)d->H, (unsigned)d->B);
  if (step && d->o_ld % 4 == 0) {
    const size_t lds = (size_t)((3 * d->dk + 3) / 4 * 4 + 1024) * 4;
    if (y16) hipLaunchKernelGGL((gated_step_kernel<uint16_t, uint16_t>), per, dim3(256), lds, st, a, s16, fs);
    else if (bf) hipLaunchKernelGGL((gated_step_kernel<float, uint16_t>), per, dim3(256), lds, st, a, s32, fs);
    else hipLaunchKernelGGL((gated_step_kernel<float, float>), per, dim3(256), lds, st, a, s32, fs);
    TNX_CHECK_LAUNCH("gated_step");
    return TNX_OK;
  }
  TNX_REQUIRE(!d->norm_w, "gated_state: output rows must be multiples of four");
  // finished bf16 rows beside finished gates, or fp32 rows throughout
  const bool plain = y16 && ys <= 1 && fsp <= 1 && d->T * (d->y.ld > d->f.ld ? d->y.ld : d->f.ld) < ((int64_t)1 << 31);
  const bool aligned = (plain || !y16 || ys > 1) && (d->y.ld | d->y.plane | d->f.ld | d->f.plane | d->q_off | d->v_off | d->f_off) % 8 == 0;
  if (bf && d->T > 1 && aligned && d->dk % 8 == 0 && d->dk <= 256 && d->dv % 8 == 0 && d->T < (1 << 30)) {
    a.span = span_tokens(d->B, d->T, d->H);
    a.n_spans = (int)cdiv(d->T, a.span);
    a.ws = d->ws;
    TNX_REQUIRE(a.n_spans == 1 || d->ws, "gated_state: a long prompt needs the workspace of tnx_gated_state_ws_bytes");
    return plain ? launch_chunk_any(st, a, s16, fs) : launch_chunk_any(st, a, s32, fs);
  }
  const size_t lds = (size_t)3 * d->dk * 4;
  if (y16) hipLaunchKernelGGL(gated_any_kernel<uint16_t>, per, dim3(256), lds, st, a, s16, fs);
  else hipLaunchKernelGGL(gated_any_kernel<float>, per, dim3(256), lds, st, a, s32, fs);
  TNX_CHECK_LAUNCH("gated_any");
  return TNX_OK;
}
