// Matrix memory with exponential gates (the mLSTM cell of xLSTM): per head a matrix state S [dk, dv], a sum of keys
// n [dk] and a running maximum m of the gates' logarithms, all fp32:
//   m' = max(f + m, i),   S' = e^(f + m - m') S + e^(i - m') k v^T,   n' = e^(f + m - m') n + e^(i - m') k,
//   o = S'^T q / (max(|n' . q|, e^(-m')) + 1e-6),
// with i = cap tanh(. / cap) and f = log sigmoid(cap tanh(. / cap)) of two fp32 columns per head.  All three begin at zero with
// a sequence's first column.
//
//   memory_chunk_kernel   prompts: 64 tokens at a time on MFMAs; a long prompt is cut into spans that run in
//                         parallel, their start states formed by a scan over spans
//   memory_step_kernel    one token per sequence: one pass over the state
//   memory_any_kernel     any sizes and fp32: token by token
#include <string.h>

#include <mutex>

#include "decoder.h"

namespace {

constexpr float kLog2e = 1.4426950408889634f;
constexpr float kFloor = 1e-6f;

struct MemoryArgs {
  int64_t B, T;
  int H, dk, dv;
  float q_scale, cap;
  int64_t q_off, k_off, v_off, i_off, f_off;
  const float* bias_i;     // [H]
  const float* bias_f;     // [H]
  const int32_t* starts;
  const int32_t* col_ptr;
  float* state;            // [B, H, dk, dv]
  float* sum;              // [B, H, dk]
  float* top;              // [B, H]
  float* o;
  int64_t o_ld;
  // chunk kernel
  int n_spans, span;       // span: tokens, a multiple of 64
  float* ws;               // [B, H, n_spans][dk dv + dk + 4]: state, sum, maximum at the end, decay (log2), maximum at the start
};

__device__ __forceinline__ float log_input(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float log_forget(float z, float cap) {
  const float y = cap * tanhf(z / cap);
  return fminf(y, 0.f) - log1pf(expf(-fabsf(y)));
}
__device__ __forceinline__ float sum256(float v, float* red) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return red[0] + red[1] + red[2] + red[3];
}

template <typename T>
__global__ __launch_bounds__(256) void memory_any_kernel(const MemoryArgs a, const RowSrc<T> src, const RowSrc<float> gates) {
  extern __shared__ float sm[];   // q [dk], k [dk], n [dk]
  __shared__ float red[4];
  const int h = blockIdx.x, tid = threadIdx.x;
  const int64_t b = blockIdx.y;
  const int col0 = *a.col_ptr, start = a.starts[b];
  float* S = a.state + (b * a.H + h) * (int64_t)a.dk * a.dv;
  float* n = sm + 2 * a.dk;
  bool fresh = col0 <= start;     // no token of this sequence has run yet
  float m = fresh ? 0.f : a.top[b * a.H + h];
  for (int i = tid; i < a.dk; i += 256) n[i] = fresh ? 0.f : a.sum[(b * a.H + h) * a.dk + i];
  const float bi = a.bias_i[h], bf = a.bias_f[h];
  for (int64_t t = max(0, start - col0); t < a.T; ++t) {
    const int64_t row = b * a.T + t;
    const float li = log_input(gates.get(row, a.i_off + h) + bi, a.cap), lf = log_forget(gates.get(row, a.f_off + h) + bf, a.cap);
    const float mn = fmaxf(lf + m, li), keep = expf(lf + m - mn), add = expf(li - mn);
    m = mn;
    __syncthreads();
    float dot = 0.f;
    for (int i = tid; i < a.dk; i += 256) {
      const float q = src.get(row, a.q_off + (int64_t)h * a.dk + i) * a.q_scale, k = src.get(row, a.k_off + (int64_t)h * a.dk + i);
      sm[i] = q;
      sm[a.dk + i] = k;
      n[i] = keep * n[i] + add * k;
      dot += n[i] * q;
    }
    const float den = fmaxf(fabsf(sum256(dot, red)), expf(-m)) + kFloor;
    for (int p = tid; p < a.dv; p += 256) {
      const float v = add * src.get(row, a.v_off + (int64_t)h * a.dv + p);
      float acc = 0.f;
#pragma unroll 8
      for (int i = 0; i < a.dk; ++i) {
        const int64_t at = (int64_t)i * a.dv + p;
        const float s = (fresh ? 0.f : keep * S[at]) + sm[a.dk + i] * v;
        S[at] = s;
        acc += sm[i] * s;
      }
      a.o[row * a.o_ld + (int64_t)h * a.dv + p] = acc / den;
    }
    fresh = false;
  }
  if (!fresh) {
    for (int i = tid; i < a.dk; i += 256) a.sum[(b * a.H + h) * a.dk + i] = n[i];
    if (tid == 0) a.top[b * a.H + h] = m;
  }
  // rows in front of the sequence: defined values for the norms behind
  for (int64_t t = 0; t < min((int64_t)max(0, start - col0), a.T); ++t)
    for (int p = tid; p < a.dv; p += 256) a.o[(b * a.T + t) * a.o_ld + (int64_t)h * a.dv + p] = 0.f;
}

// One token: a thread owns four value columns and every NG-th row of the state.
template <typename T>
__global__ __launch_bounds__(256) void memory_step_kernel(const MemoryArgs a, const RowSrc<T> src, const RowSrc<float> gates) {
  extern __shared__ __align__(16) float sm[];   // q [dk], k [dk], then the partial outputs [256][4]
  __shared__ float red[4];
  const int h = blockIdx.x, tid = threadIdx.x;
  const int64_t b = blockIdx.y;
  const int nc = a.dv / 4, ng = 256 / nc, grp = tid / nc, c = tid % nc;
  const bool fresh = *a.col_ptr <= a.starts[b], mine = grp < ng;
  f32x4* part = reinterpret_cast<f32x4*>(sm + (2 * a.dk + 3) / 4 * 4);
  f32x4* S = reinterpret_cast<f32x4*>(a.state + (b * a.H + h) * (int64_t)a.dk * a.dv);
  // the first rows of the state are on their way while q, k and v arrive
  constexpr int PF = 8;
  f32x4 s[PF];
#pragma unroll
  for (int u = 0; u < PF; ++u) {
    const int i = grp + u * ng;
    s[u] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (mine && i < a.dk && !fresh) s[u] = __builtin_nontemporal_load(&S[(int64_t)i * nc + c]);
  }
  const float m = fresh ? 0.f : a.top[b * a.H + h];
  const float li = log_input(gates.get(b, a.i_off + h) + a.bias_i[h], a.cap), lf = log_forget(gates.get(b, a.f_off + h) + a.bias_f[h], a.cap);
  const float mn = fmaxf(lf + m, li), keep = fresh ? 0.f : expf(lf + m - mn), add = expf(li - mn);
  float dot = 0.f;
  for (int i = tid; i < a.dk; i += 256) {
    const float q = src.get(b, a.q_off + (int64_t)h * a.dk + i) * a.q_scale, k = src.get(b, a.k_off + (int64_t)h * a.dk + i);
    float* n = a.sum + (b * a.H + h) * a.dk + i;
    sm[i] = q;
    sm[a.dk + i] = k;
    const float nn = (fresh ? 0.f : keep * *n) + add * k;
    *n = nn;
    dot += nn * q;
  }
  f32x4 v = f32x4{0.f, 0.f, 0.f, 0.f}, acc = v;
  if (mine)
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = add * src.get(b, a.v_off + (int64_t)h * a.dv + c * 4 + e);
  const float den = fmaxf(fabsf(sum256(dot, red)), expf(-mn)) + kFloor;   // (its barriers also publish q and k)
  if (tid == 0) a.top[b * a.H + h] = mn;
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
          const f32x4 w = keep * s[u] + sm[a.dk + i] * v;
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
    for (int e = 0; e < 4; ++e) o[e] = t[e] / den;
  }
}

constexpr int kChunk = 64, kTLD = kChunk + 8;
constexpr float kNone = -1.0e30f, kMasked = -2.0e30f;   // no maximum yet; a token outside the sequence
constexpr size_t memory_smem_bytes(int kt) {
  // q, k [64][dk + 8]; k^T [dk][72]; v^T [128][72] (bf16); six tables of 64, n [dk], four tables of 64 per wave
  return (size_t)(2 * kChunk * (kt * 32 + 8) + kt * 32 * kTLD + 128 * kTLD) * 2 + (6 * 64 + kt * 32 + 4 * 64) * 4;
}
__device__ __forceinline__ u32x4 fetch8(const RowSrc<uint16_t>& s, int64_t row, int64_t col) {
  if (s.split <= 1) return *reinterpret_cast<const u32x4*>(s.y + row * s.ld + col);
  float f[8];
  get8(s, row, col, f);
  return u32x4{pack2bf(f[0], f[1]), pack2bf(f[2], f[3]), pack2bf(f[4], f[5]), pack2bf(f[6], f[7])};
}

// A work-group takes one span of one (row, head) and up to 128 value columns; wave w keeps the state of columns
// 32 w .. + 31 in its accumulators (fp32), a thread one element of the sum of keys.  Per chunk of 64 tokens, in log2
// units, with L the running sum of f from the chunk's start, m the maximum in front of it and
//   c_j = i_j - L_j,   M_t = max(m, c_1, .., c_t)        (so that the maximum behind token t is L_t + M_t):
//   num_t = 2^(m - M_t) q_t S + sum_{j <= t} 2^(c_j - M_t) (q_t . k_j) v_j,   n . q likewise,
//   S = 2^(m - M_64) S + sum_j k_j (2^(c_j - M_64) v_j)^T.
// No weight exceeds one and no decay is ever divided by.  The accumulator layout of S is, in a permuted order of
// the head dimension that q's fragments follow, the B operand of q S; likewise the scores (computed transposed) are the
// A operand of the product with v.  fp32 operands (S, weighted scores, weighted v) enter as a high and a low bf16
// part.  STATES: only the span's own contribution is formed (into ws), from no maximum at all.
template <int KT, bool STATES>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, KT <= 4 ? 2 : 1))) void memory_chunk_kernel(const MemoryArgs a, const RowSrc<uint16_t> src,
                                                                                                                     const RowSrc<float> gates) {
  constexpr int DK = KT * 32, QLD = DK + 8;
  extern __shared__ __align__(16) unsigned char smem[];
  uint16_t* qs = reinterpret_cast<uint16_t*>(smem);
  uint16_t* ks = qs + kChunk * QLD;
  uint16_t* ktr = ks + kChunk * QLD;
  uint16_t* vt = ktr + DK * kTLD;
  float* tc = reinterpret_cast<float*>(vt + 128 * kTLD);   // c_j
  float* tm = tc + 64;                                     // M_t
  float* te = tc + 128;                                    // 2^(m - M_t), times the query's scale
  float* tw = tc + 192;                                    // 2^(c_j - M_64)
  float* tf = tc + 256;                                    // 2^-(L_t + M_t)
  float* tq = tc + 320;                                    // n . q_t, n in front of the chunk
  float* ns = tc + 384;                                    // n
  const int tid = threadIdx.x, lane = tid & 63, l32 = lane & 31, lh = lane >> 5;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  float* td = ns + DK + wave * 64;                         // 1 / denominator of token t
  const int span = blockIdx.x % a.n_spans, slice = blockIdx.x / a.n_spans;
  const int h = blockIdx.y;
  const int64_t b = blockIdx.z, bh = b * a.H + h;
  if (STATES && span == a.n_spans - 1) return;             // nothing starts from the last span's state
  const int64_t rec = (int64_t)a.dk * a.dv + a.dk + 4;
  float* wrec = a.ws + (bh * a.n_spans + span) * rec;      // (read and written only with several spans)
  const int col0 = *a.col_ptr, start = a.starts[b];
  const int dvw = slice * 128 + wave * 32;                 // this wave's first value column
  const bool active = dvw < a.dv;
  const int t_begin = span * a.span, t_end = min((int)a.T, t_begin + a.span);
  const int dcol = dvw + l32;                              // this lane's value column
  const bool dok = dcol < a.dv;
  const float bi = a.bias_i[h], bf = a.bias_f[h];

  float m = STATES ? kNone : 0.f, decay = 0.f, nreg = 0.f;   // (log2 units)
  f32x16 S[KT];
  {
    const float* init = nullptr;
    if (!STATES) {
      if (a.n_spans > 1) {
        init = wrec;
        m = wrec[rec - 2];
        if (tid < a.dk) nreg = wrec[(int64_t)a.dk * a.dv + tid];
      } else if (col0 > start) {
        init = a.state + bh * (int64_t)a.dk * a.dv;
        m = a.top[bh] * kLog2e;
        if (tid < a.dk) nreg = a.sum[bh * a.dk + tid];
      }
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
  constexpr int VI = 2;                                                   // 32 pairs x 16 runs of v
  u32x4 qr[QI][2], kr[QI][2], vr[VI][2];
  float i_raw = 0.f, f_raw = 0.f;
  const u32x4 zero = u32x4{0, 0, 0, 0};
  auto fetch = [&](int t0) {
#pragma unroll
    for (int c = 0; c < QI; ++c) {
      const int it = c * 256 + tid, pr = it / (DK / 8), ch = it % (DK / 8);
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int t = t0 + 2 * pr + e;
        const bool ok = pr < 32 && ch * 8 < a.dk && t < t_end && col0 + t >= start;
        const int64_t at = (int64_t)h * a.dk + ch * 8;
        kr[c][e] = ok ? fetch8(src, b * a.T + t, a.k_off + at) : zero;
        if (!STATES) qr[c][e] = ok ? fetch8(src, b * a.T + t, a.q_off + at) : zero;
      }
    }
#pragma unroll
    for (int c = 0; c < VI; ++c) {
      const int it = c * 256 + tid, pr = it / 16, d = slice * 128 + (it % 16) * 8;
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int t = t0 + 2 * pr + e;
        const bool ok = d < a.dv && t < t_end && col0 + t >= start;
        vr[c][e] = ok ? fetch8(src, b * a.T + t, a.v_off + (int64_t)h * a.dv + d) : zero;
      }
    }
    const int t = t0 + lane;
    if (t < t_end) {
      i_raw = gates.get(b * a.T + t, a.i_off + h);
      f_raw = gates.get(b * a.T + t, a.f_off + h);
    }
  };
  // two tokens' runs of eight -> eight words (token, next token)
  auto pair_word = [](const u32x4& x, const u32x4& y, int j) -> uint32_t {
    return __builtin_amdgcn_perm(y[j >> 1], x[j >> 1], (j & 1) ? 0x07060302u : 0x05040100u);
  };

  // chunks wholly in front of the sequence change nothing
  int t0 = t_begin;
  if (start > col0) t0 = max(t_begin, t_begin + (start - col0 - t_begin) / kChunk * kChunk);
  if (!STATES && dok)
    for (int t = t_begin + lh; t < min(t0, t_end); t += 2) a.o[(b * a.T + t) * a.o_ld + (int64_t)h * a.dv + dcol] = 0.f;
  if (t0 < t_end) fetch(t0);
  for (; t0 < t_end; t0 += kChunk) {
    const int n = min(kChunk, t_end - t0);
    __syncthreads();    // the readers of the chunk before are done
#pragma unroll
    for (int c = 0; c < QI; ++c) {
      const int it = c * 256 + tid, pr = it / (DK / 8), ch = it % (DK / 8);
      if (pr >= 32) continue;
      if (!STATES) {
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          *reinterpret_cast<u32x4*>(&qs[(2 * pr + e) * QLD + ch * 8]) = qr[c][e];
          *reinterpret_cast<u32x4*>(&ks[(2 * pr + e) * QLD + ch * 8]) = kr[c][e];
        }
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) *reinterpret_cast<uint32_t*>(&ktr[(ch * 8 + j) * kTLD + 2 * pr]) = pair_word(kr[c][0], kr[c][1], j);
    }
#pragma unroll
    for (int c = 0; c < VI; ++c) {
      const int it = c * 256 + tid, pr = it / 16, ch = it % 16;
#pragma unroll
      for (int j = 0; j < 8; ++j) *reinterpret_cast<uint32_t*>(&vt[(ch * 8 + j) * kTLD + 2 * pr]) = pair_word(vr[c][0], vr[c][1], j);
    }
    if (!STATES && tid < DK) ns[tid] = nreg;
    // the gates; tokens outside the sequence neither decay nor add
    const bool real = lane < n && col0 + t0 + lane >= start;
    float L = real ? log_forget(f_raw + bf, a.cap) * kLog2e : 0.f;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float v = __shfl_up(L, o, 64);
      if (lane >= o) L += v;
    }
    const float cj = real ? log_input(i_raw + bi, a.cap) * kLog2e - L : kMasked;
    float M = fmaxf(cj, m);
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float v = __shfl_up(M, o, 64);
      if (lane >= o) M = fmaxf(M, v);
    }
    const float Ln = __shfl(L, 63, 64), Mn = __shfl(M, 63, 64), keep = __builtin_amdgcn_exp2f(m - Mn);
    if (wave == 0) {
      tc[lane] = cj;
      tm[lane] = M;
      te[lane] = __builtin_amdgcn_exp2f(m - M) * a.q_scale;
      tw[lane] = __builtin_amdgcn_exp2f(cj - Mn);
      tf[lane] = __builtin_amdgcn_exp2f(-(L + M));
    }
    decay += Ln;
    m = Ln + Mn;
    __syncthreads();
    if (t0 + kChunk < t_end) fetch(t0 + kChunk);
    if constexpr (!STATES) {
      // n . q: four threads per token
      const int tok = tid >> 2;
      float dot = 0.f;
#pragma unroll
      for (int i = 0; i < DK / 4; i += 8) {
        const int d = (tid & 3) * (DK / 4) + i;
        const u32x4 qv = *reinterpret_cast<const u32x4*>(&qs[tok * QLD + d]);
#pragma unroll
        for (int r = 0; r < 4; ++r) dot += bflo(qv[r]) * ns[d + 2 * r] + bfhi(qv[r]) * ns[d + 2 * r + 1];
      }
      dot += __shfl_xor(dot, 1, 64);
      dot += __shfl_xor(dot, 2, 64);
      if ((tid & 3) == 0) tq[tok] = dot;
      __syncthreads();
    }
    if (tid < DK) {
      float s = 0.f;
#pragma unroll
      for (int j = 0; j < kChunk; j += 8) {
        const u32x4 kv = *reinterpret_cast<const u32x4*>(&ktr[tid * kTLD + j]);
#pragma unroll
        for (int r = 0; r < 4; ++r) s += bflo(kv[r]) * tw[j + 2 * r] + bfhi(kv[r]) * tw[j + 2 * r + 1];
      }
      nreg = keep * nreg + s;
    }
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
          u32x4 sh, sl;
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            uint32_t hi, lo;
            split2(S[kt][8 * s + 2 * r], S[kt][8 * s + 2 * r + 1], hi, lo);
            sh[r] = hi;
            sl[r] = lo;
          }
#pragma unroll
          for (int qt = 0; qt < 2; ++qt) {
            const uint16_t* p = &qs[(qt * 32 + l32) * QLD + kt * 32 + 16 * s + 4 * lh];
            const u32x2 p0 = *reinterpret_cast<const u32x2*>(p), p1 = *reinterpret_cast<const u32x2*>(p + 8);
            const u32x4 af = {p0[0], p0[1], p1[0], p1[1]};
            O[qt] = mfma32(af, sh, O[qt]);
            O[qt] = mfma32(af, sl, O[qt]);
          }
        }
#pragma unroll
      for (int qt = 0; qt < 2; ++qt)
#pragma unroll
        for (int bb = 0; bb < 4; ++bb) {
          const f32x4 w = *reinterpret_cast<const f32x4*>(&te[qt * 32 + 8 * bb + 4 * lh]);
#pragma unroll
          for (int e = 0; e < 4; ++e) O[qt][4 * bb + e] *= w[e];
        }
      // inside the chunk
#pragma unroll
      for (int qt = 0; qt < 2; ++qt) {
        const int tq_ = qt * 32 + l32;
        const float Mq = tm[tq_];
        float rs = 0.f;
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
          for (int bb = 0; bb < 4; ++bb) {
            const int k0 = jt * 32 + 8 * bb + 4 * lh;
            const f32x4 ck = *reinterpret_cast<const f32x4*>(&tc[k0]);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              const float w = __builtin_amdgcn_exp2f(fminf(ck[e] - Mq, 0.f)) * a.q_scale;
              st[4 * bb + e] = k0 + e <= tq_ ? st[4 * bb + e] * w : 0.f;
              rs += st[4 * bb + e];
            }
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
            const u32x4 vf = {p0[0], p0[1], p1[0], p1[1]};
            O[qt] = mfma32(ah, vf, O[qt]);
            O[qt] = mfma32(al, vf, O[qt]);
          }
        }
        rs += __shfl_xor(rs, 32, 64);
        if (lh == 0) td[tq_] = 1.0f / (fmaxf(fabsf(te[tq_] * tq[tq_] + rs), tf[tq_]) + kFloor);
      }
      if (dok)
#pragma unroll
        for (int qt = 0; qt < 2; ++qt)
#pragma unroll
          for (int bb = 0; bb < 4; ++bb) {
            const int r0 = qt * 32 + 8 * bb + 4 * lh;
            const f32x4 w = *reinterpret_cast<const f32x4*>(&td[r0]);
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (r0 + e < n) a.o[(b * a.T + t0 + r0 + e) * a.o_ld + (int64_t)h * a.dv + dcol] = O[qt][4 * bb + e] * w[e];
          }
    }
    // the state behind this chunk
    u32x4 vh[4], vl[4];
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const u32x4 xv = *reinterpret_cast<const u32x4*>(&vt[(wave * 32 + l32) * kTLD + 16 * s + 8 * lh]);
      const f32x4 w0 = *reinterpret_cast<const f32x4*>(&tw[16 * s + 8 * lh]), w1 = *reinterpret_cast<const f32x4*>(&tw[16 * s + 8 * lh + 4]);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float wa = r < 2 ? w0[2 * r] : w1[2 * r - 4], wb = r < 2 ? w0[2 * r + 1] : w1[2 * r - 3];
        uint32_t hi, lo;
        split2(bflo(xv[r]) * wa, bfhi(xv[r]) * wb, hi, lo);
        vh[s][r] = hi;
        vl[s][r] = lo;
      }
    }
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
#pragma unroll
      for (int i = 0; i < 16; ++i) S[kt][i] *= keep;
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        const u32x4 kf = *reinterpret_cast<const u32x4*>(&ktr[(kt * 32 + l32) * kTLD + 16 * s + 8 * lh]);
        S[kt] = mfma32(kf, vh[s], S[kt]);
        S[kt] = mfma32(kf, vl[s], S[kt]);
      }
    }
  }
  float *dst = nullptr, *ndst = nullptr;
  if (STATES) {
    dst = wrec;
    ndst = wrec + (int64_t)a.dk * a.dv;
    if (slice == 0 && tid == 0) {
      wrec[rec - 4] = m;
      wrec[rec - 3] = decay;
    }
  } else if (span == a.n_spans - 1 && (a.T + col0 > start)) {
    dst = a.state + bh * (int64_t)a.dk * a.dv;
    ndst = a.sum + bh * a.dk;
    if (slice == 0 && tid == 0) a.top[bh] = m * (1.0f / kLog2e);
  }
  if (!dst) return;
  if (slice == 0 && tid < a.dk) ndst[tid] = nreg;
  if (dok)
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int r = kt * 32 + 8 * (i >> 2) + 4 * lh + (i & 3);
        if (r < a.dk) dst[(int64_t)r * a.dv + dcol] = S[kt][i];
      }
}

// the spans' own contributions -> what each span starts from, in place
__global__ __launch_bounds__(256) void memory_scan_kernel(const MemoryArgs a) {
  const int64_t nS = (int64_t)a.dk * a.dv, n = nS + a.dk, rec = n + 4, i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  const int64_t bh = (int64_t)blockIdx.z * a.H + blockIdx.y;
  if (i >= n) return;
  const bool fresh = *a.col_ptr <= a.starts[blockIdx.z];
  float cur = fresh ? 0.f : i < nS ? a.state[bh * nS + i] : a.sum[bh * a.dk + i - nS];
  float m = fresh ? 0.f : a.top[bh] * kLog2e;
  float* p = a.ws + bh * a.n_spans * rec;
  for (int s = 0; s < a.n_spans; ++s, p += rec) {
    const bool more = s + 1 < a.n_spans;
    const float own = more ? p[i] : 0.f, top = more ? p[rec - 4] : kNone, f = more ? p[rec - 3] : 0.f;
    p[i] = cur;
    if (i == 0) p[rec - 2] = m;
    const float mn = fmaxf(f + m, top);
    cur = __builtin_amdgcn_exp2f(f + m - mn) * cur + __builtin_amdgcn_exp2f(top - mn) * own;
    m = mn;
  }
}

template <int KT>
int launch_chunk(hipStream_t st, const MemoryArgs& a, const RowSrc<uint16_t>& src, const RowSrc<float>& gates) {
  static std::once_flag once;
  static hipError_t e = hipSuccess;
  constexpr size_t kSmem = memory_smem_bytes(KT);
  std::call_once(once, [] {
    e = hipFuncSetAttribute(reinterpret_cast<const void*>(&memory_chunk_kernel<KT, false>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kSmem);
    if (e == hipSuccess)
      e = hipFuncSetAttribute(reinterpret_cast<const void*>(&memory_chunk_kernel<KT, true>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kSmem);
  });
  if (e != hipSuccess) {
    tnx_set_error("memory: cannot raise the dynamic LDS limit: %s", hipGetErrorString(e));
    return TNX_ELAUNCH;
  }
  const dim3 grid((unsigned)(a.n_spans * cdiv(a.dv, 128)), (unsigned)a.H, (unsigned)a.B);
  if (a.n_spans > 1) {
    hipLaunchKernelGGL((memory_chunk_kernel<KT, true>), grid, dim3(256), kSmem, st, a, src, gates);
    hipLaunchKernelGGL(memory_scan_kernel, dim3((unsigned)cdiv((int64_t)a.dk * (a.dv + 1), 256), (unsigned)a.H, (unsigned)a.B), dim3(256), 0, st, a);
  }
  hipLaunchKernelGGL((memory_chunk_kernel<KT, false>), grid, dim3(256), kSmem, st, a, src, gates);
  TNX_CHECK_LAUNCH("memory_chunk");
  return TNX_OK;
}

// work-groups of a prompt pass that fill the device; shorter spans cost state traffic
int span_tokens(int64_t B, int64_t T, int H, int dv) {
  const int64_t per = B * H * cdiv(dv, 128);
  int64_t spans = per >= 256 ? 1 : cdiv(512, per);
  int64_t span = cdiv(cdiv(T, spans), kChunk) * kChunk;
  if (span < 2 * kChunk) span = 2 * kChunk;
  return (int)span;
}

}  // namespace

extern "C" size_t tnx_memory_ws_bytes(int64_t B, int64_t T, int H, int dk, int dv) {
  if (T <= 1 || B <= 0 || H <= 0 || dk <= 0 || dv <= 0) return 0;
  const int64_t spans = cdiv(T, span_tokens(B, T, H, dv));
  return spans > 1 ? (size_t)(B * H * spans) * ((size_t)dk * (size_t)dv + dk + 4) * 4 : 0;
}

extern "C" int tnx_memory(void* stream, const tnx_memory_desc* d) {
  TNX_REQUIRE(d, "memory: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->T > 0 && d->H > 0 && d->dk > 0 && d->dv > 0, "memory: bad shape");
  TNX_REQUIRE(d->bias_i && d->bias_f && d->starts && d->col_ptr && d->state && d->sum && d->top && d->o && src_given(d->y) && src_given(d->gates), "memory: null pointer");
  TNX_REQUIRE(d->o_ld >= (int64_t)d->H * d->dv && d->dk <= 4096 && d->cap > 0.f, "memory: short output rows, a head size above 4096 or no cap");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "memory: bad dtype %d", d->dtype);
  TNX_REQUIRE(d->B <= 65535 && d->H <= 65535, "memory: too many rows or heads");
  MemoryArgs a;
  memset(&a, 0, sizeof(a));
  a.B = d->B; a.T = d->T; a.H = d->H; a.dk = d->dk; a.dv = d->dv; a.q_scale = d->q_scale; a.cap = d->cap; a.q_off = d->q_off; a.k_off = d->k_off;
  a.v_off = d->v_off; a.i_off = d->i_off; a.f_off = d->f_off; a.bias_i = d->bias_i; a.bias_f = d->bias_f; a.starts = d->starts; a.col_ptr = d->col_ptr;
  a.state = d->state; a.sum = d->sum; a.top = d->top; a.o = d->o; a.o_ld = d->o_ld;
  hipStream_t st = as_stream(stream);
  const bool bf = d->dtype == TNX_BF16;
  const RowSrc<uint16_t> s16{(const uint16_t*)d->y.y, d->y.ws, d->y.split_k, d->y.plane, d->y.ld};
  const RowSrc<float> s32{(const float*)d->y.y, d->y.ws, d->y.split_k, d->y.plane, d->y.ld};
  const RowSrc<float> gates{(const float*)d->gates.y, d->gates.ws, d->gates.split_k, d->gates.plane, d->gates.ld};
  const dim3 per((unsigned)d->H, (unsigned)d->B);
  if (d->T == 1 && d->dv % 4 == 0 && d->dv <= 1024) {
    const size_t lds = (size_t)((2 * d->dk + 3) / 4 * 4 + 1024) * 4;
    if (bf) hipLaunchKernelGGL(memory_step_kernel<uint16_t>, per, dim3(256), lds, st, a, s16, gates);
    else hipLaunchKernelGGL(memory_step_kernel<float>, per, dim3(256), lds, st, a, s32, gates);
    TNX_CHECK_LAUNCH("memory_step");
    return TNX_OK;
  }
  if (bf && d->T > 1 && d->dk % 8 == 0 && d->dk <= 256 && d->dv % 8 == 0 && (d->q_off | d->k_off | d->v_off) % 8 == 0 && d->y.ld % 8 == 0 &&
      (d->y.split_k <= 1 || d->y.plane % 8 == 0) && d->T < (1 << 30)) {
    a.span = span_tokens(d->B, d->T, d->H, d->dv);
    a.n_spans = (int)cdiv(d->T, a.span);
    a.ws = d->ws;
    TNX_REQUIRE(a.n_spans == 1 || d->ws, "memory: a long prompt needs the workspace of tnx_memory_ws_bytes");
    if (d->dk <= 32) return launch_chunk<1>(st, a, s16, gates);
    if (d->dk <= 64) return launch_chunk<2>(st, a, s16, gates);
    if (d->dk <= 128) return launch_chunk<4>(st, a, s16, gates);
    return launch_chunk<8>(st, a, s16, gates);
  }
  const size_t lds = (size_t)3 * d->dk * 4;
  if (bf) hipLaunchKernelGGL(memory_any_kernel<uint16_t>, per, dim3(256), lds, st, a, s16, gates);
  else hipLaunchKernelGGL(memory_any_kernel<float>, per, dim3(256), lds, st, a, s32, gates);
  TNX_CHECK_LAUNCH("memory_any");
  return TNX_OK;
}
