// State-space duality layers (per head a matrix state S [N, P] in fp32, decays that depend on the token):
//   dt = softplus(raw + bias_h),   S_t = exp(-exp(A_h) dt) S_(t-1) + dt B_t x_t^T,   y_t = S_t^T C_t + D_h x_t,
// with x, B and C behind a causal convolution per channel and silu; B and C are shared by the heads of a
// group.  y leaves in fp32 [rows, H * P]; the state [B, H, N, P] is read (from a sequence's first column
// on: taken as zero) and written back.  The convolution's inputs of the last columns live in a ring
// [B, slots, channels], slot = column % slots.
//
//   short_conv_kernel / _vec_kernel   convolution + silu of many tokens
//   ring_write_kernel                 the last columns' rows into a ring
//   ssd_chunk_kernel                  prompts: 64 tokens at a time on MFMAs; a long prompt is cut into spans
//                                     that run in parallel, their start states formed by a scan over spans
//   ssd_step_kernel                   one token per sequence: convolution, one pass over the state, ring write
//   ssd_any_kernel                    any sizes and fp32: token by token
#include <string.h>

#include <mutex>

#include "decoder.h"

namespace {

__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
constexpr float kLog2e = 1.4426950408889634f;

// ---- short convolution --------------------------------------------------------------------------
struct ConvArgs {
  int64_t B, T, C, off, out_ld;
  int taps, slots;
  const float* w;          // [taps, C], the last row belongs to the current token
  const float* bias;       // [C]
  const void* ring;        // [B, slots, C]
  const int32_t* starts;
  const int32_t* col_ptr;
  void* out;
};

template <typename T>
__global__ __launch_bounds__(256) void short_conv_kernel(const ConvArgs a, const RowSrc<T> src) {
  const int64_t c = (int64_t)blockIdx.x * 256 + threadIdx.x, row = (int64_t)blockIdx.z * 32768 + blockIdx.y;
  if (c >= a.C || row >= a.B * a.T) return;
  const int64_t b = row / a.T, t = row % a.T;
  const int col0 = *a.col_ptr, start = a.starts[b];
  const T* ring = reinterpret_cast<const T*>(a.ring) + b * a.slots * a.C;
  float v = a.bias[c];
  for (int j = a.taps - 1; j >= 0; --j) {
    const int64_t col = col0 + t - j;
    if (col < start) continue;
    const float u = t >= j ? src.get(row - j, a.off + c) : ld_elem(ring, (col % a.slots) * a.C + c);
    v += a.w[(int64_t)(a.taps - 1 - j) * a.C + c] * u;
  }
  st_elem(reinterpret_cast<T*>(a.out), row * a.out_ld + c, silu_f32(v));
}

// A thread takes eight channels and up to kConvRun tokens; the inputs of the tokens before stay in registers.
constexpr int kConvRun = 16;
template <int TAPS, typename T>
__global__ __launch_bounds__(256) void short_conv_vec_kernel(const ConvArgs a, const RowSrc<T> src, int run) {
  const int nch = (int)(a.C / 8), runs = (int)((a.T + run - 1) / run);
  const int64_t item = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (item >= a.B * runs * nch) return;
  const int64_t c = item % nch * 8, b = item / nch / runs, t0 = item / nch % runs * run;
  const int col0 = *a.col_ptr, start = a.starts[b];
  const RowSrc<T> ring{reinterpret_cast<const T*>(a.ring) + b * a.slots * a.C, nullptr, 1, 0, a.C};
  const RowSrc<float> wsrc{a.w, nullptr, 1, 0, a.C}, bsrc{a.bias, nullptr, 1, 0, 0};
  float w[TAPS][8], bias[8], u[TAPS][8];
#pragma unroll
  for (int k = 0; k < TAPS; ++k) get8(wsrc, k, c, w[k]);
  get8(bsrc, 0, c, bias);
  auto input = [&](int64_t t, float (&f)[8]) {
    const int64_t col = col0 + t;
    if (col < start) {
#pragma unroll
      for (int i = 0; i < 8; ++i) f[i] = 0.f;
    } else if (t >= 0) {
      get8(src, b * a.T + t, a.off + c, f);
    } else {
      get8(ring, col % a.slots, c, f);
    }
  };
#pragma unroll
  for (int k = 0; k + 1 < TAPS; ++k) input(t0 - (TAPS - 1) + k, u[k]);
  const int64_t t1 = min(a.T, t0 + run);
  for (int64_t t = t0; t < t1; ++t) {
    input(t, u[TAPS - 1]);
    float v[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      v[i] = bias[i];
#pragma unroll
      for (int k = 0; k < TAPS; ++k) v[i] += w[k][i] * u[k][i];
      v[i] = silu_f32(v[i]);
    }
    put8(reinterpret_cast<T*>(a.out) + (b * a.T + t) * a.out_ld + c, v);
#pragma unroll
    for (int k = 0; k + 1 < TAPS; ++k)
#pragma unroll
      for (int i = 0; i < 8; ++i) u[k][i] = u[k + 1][i];
  }
}

// ring[b, (col + t) % slots, :] = rows of the last min(T, slots) tokens
template <typename T>
__global__ __launch_bounds__(256) void ring_write_kernel(int64_t Tn, int64_t C, int64_t off, int slots, const int32_t* col_ptr,
                                                         int64_t t0, const RowSrc<T> src, T* ring) {
  const int64_t c = (int64_t)blockIdx.x * 256 + threadIdx.x, b = blockIdx.z, t = Tn - 1 - blockIdx.y;
  if (c >= C) return;
  st_elem(ring, (b * slots + (*col_ptr + t0 + t) % slots) * C + c, src.get(b * Tn + t, off + c));
}

// ---- the recurrence -----------------------------------------------------------------------------
struct SsdArgs {
  int64_t B, T;
  int H, G, N, P, hpg;     // heads, groups, state and value sizes, heads of a group
  const float* A_log;      // [H]
  const float* dt_bias;    // [H]
  const float* D;          // [H]
  const int32_t* starts;
  const int32_t* col_ptr;
  int64_t dt_off, o_ld;
  float* state;
  float* o;
  // convolved rows [B * T, u_ld]: x from 0, B from H P, C from H P + G N
  const void* u;
  int64_t u_ld;
  // step: the convolution
  int64_t c_off;
  int taps, slots;
  const float* conv_w;
  const float* conv_b;
  void* ring;
  // chunk kernel
  int n_spans, span;       // span: tokens, a multiple of 64
  int pp, slices;          // columns of a head, padded to 32; 128-column slices of a group
  float* ws;               // [B, H, n_spans, N, P], then the spans' decays [B, H, n_spans]
};

template <typename T>
__global__ __launch_bounds__(256) void ssd_any_kernel(const SsdArgs a, const RowSrc<T> src) {
  extern __shared__ float sm[];   // B [N], C [N]
  const int h = blockIdx.x, g = h / a.hpg, tid = threadIdx.x;
  const int64_t b = blockIdx.y;
  const int col0 = *a.col_ptr, start = a.starts[b];
  const float A = expf(a.A_log[h]), bias = a.dt_bias[h], Dh = a.D[h];
  const T* u = reinterpret_cast<const T*>(a.u);
  float* S = a.state + (b * a.H + h) * (int64_t)a.N * a.P;
  const int64_t inner = (int64_t)a.H * a.P;
  bool fresh = col0 <= start;     // no token of this sequence has run yet
  for (int64_t t = max(0, start - col0); t < a.T; ++t) {
    const int64_t row = b * a.T + t;
    const float dt = softplus_f32(src.get(row, a.dt_off + h) + bias), lam = expf(-A * dt);
    __syncthreads();
    for (int i = tid; i < a.N; i += 256) {
      sm[i] = ld_elem(u, row * a.u_ld + inner + (int64_t)g * a.N + i);
      sm[a.N + i] = ld_elem(u, row * a.u_ld + inner + (int64_t)(a.G + g) * a.N + i);
    }
    __syncthreads();
    for (int p = tid; p < a.P; p += 256) {
      const float x = ld_elem(u, row * a.u_ld + (int64_t)h * a.P + p);
      float acc = 0.f;
#pragma unroll 8
      for (int i = 0; i < a.N; ++i) {
        const int64_t at = (int64_t)i * a.P + p;
        const float s = (fresh ? 0.f : lam * S[at]) + dt * sm[i] * x;
        S[at] = s;
        acc += sm[a.N + i] * s;
      }
      a.o[row * a.o_ld + (int64_t)h * a.P + p] = acc + Dh * x;
    }
    fresh = false;
  }
  // rows in front of the sequence: defined values for the norms behind
  for (int64_t t = 0; t < min((int64_t)max(0, start - col0), a.T); ++t)
    for (int p = tid; p < a.P; p += 256) a.o[(b * a.T + t) * a.o_ld + (int64_t)h * a.P + p] = 0.f;
}

// One token: a thread owns four value columns and every NG-th row of the state.  The ring slot of the
// current column is written and never read here, so the work-groups of a group's heads may all read the
// group's channels while the first of them writes them.
template <typename T>
__global__ __launch_bounds__(256) void ssd_step_kernel(const SsdArgs a, const RowSrc<T> src) {
  extern __shared__ __align__(16) float sm[];   // x [P], B [N], C [N], then the partial outputs [256][4]
  const int h = blockIdx.x, g = h / a.hpg, tid = threadIdx.x;
  const int64_t b = blockIdx.y;
  const int nc = a.P / 4, ng = 256 / nc, grp = tid / nc, c = tid % nc;
  const int col = *a.col_ptr, start = a.starts[b];
  const bool fresh = col <= start, mine = grp < ng;
  f32x4* part = reinterpret_cast<f32x4*>(sm + (a.P + 2 * a.N + 3) / 4 * 4);
  f32x4* S = reinterpret_cast<f32x4*>(a.state + (b * a.H + h) * (int64_t)a.N * a.P);
  // the first rows of the state are on their way while the convolution runs
  constexpr int PF = 8;
  f32x4 s[PF];
#pragma unroll
  for (int u = 0; u < PF; ++u) {
    const int i = grp + u * ng;
    s[u] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (mine && i < a.N && !fresh) s[u] = __builtin_nontemporal_load(&S[(int64_t)i * nc + c]);
  }
  const int64_t inner = (int64_t)a.H * a.P, C = inner + 2 * (int64_t)a.G * a.N;
  T* ring = reinterpret_cast<T*>(a.ring) + b * a.slots * C;
  const int now = col % a.slots;
  const bool writes_shared = h % a.hpg == 0;
  for (int i = tid; i < a.P + 2 * a.N; i += 256) {
    const int64_t ch = i < a.P ? (int64_t)h * a.P + i
                               : i < a.P + a.N ? inner + (int64_t)g * a.N + (i - a.P) : inner + (int64_t)(a.G + g) * a.N + (i - a.P - a.N);
    float v = a.conv_b[ch];
    for (int j = a.taps - 1; j > 0; --j)
      if (col - j >= start) v += a.conv_w[(int64_t)(a.taps - 1 - j) * C + ch] * ld_elem(ring, (int64_t)((col - j) % a.slots) * C + ch);
    const float cur = src.get(b, a.c_off + ch);
    v += a.conv_w[(int64_t)(a.taps - 1) * C + ch] * cur;
    if (i < a.P || writes_shared) st_elem(ring, (int64_t)now * C + ch, cur);
    sm[i] = silu_f32(v);
  }
  const float dt = softplus_f32(src.get(b, a.dt_off + h) + a.dt_bias[h]);
  const float lam = fresh ? 0.f : expf(-expf(a.A_log[h]) * dt), Dh = a.D[h];
  __syncthreads();
  const float* Bs = sm + a.P;
  const float* Cs = Bs + a.N;
  f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
  if (mine) {
    f32x4 x;
#pragma unroll
    for (int e = 0; e < 4; ++e) x[e] = sm[c * 4 + e] * dt;
    for (int i0 = grp; i0 < a.N; i0 += PF * ng) {
      f32x4 nx[PF];
#pragma unroll
      for (int u = 0; u < PF; ++u) {
        const int i = i0 + (PF + u) * ng;
        nx[u] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (i < a.N && !fresh) nx[u] = __builtin_nontemporal_load(&S[(int64_t)i * nc + c]);
      }
#pragma unroll
      for (int u = 0; u < PF; ++u) {
        const int i = i0 + u * ng;
        if (i < a.N) {
          const f32x4 w = lam * s[u] + Bs[i] * x;
          __builtin_nontemporal_store(w, &S[(int64_t)i * nc + c]);
          acc += Cs[i] * w;
        }
        s[u] = nx[u];
      }
    }
  }
  part[tid] = acc;
  __syncthreads();
  if (tid < nc) {
    f32x4 t = part[tid];
    for (int gq = 1; gq < ng; ++gq) t += part[gq * nc + tid];
    float* o = a.o + b * a.o_ld + (int64_t)h * a.P + tid * 4;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = t[e] + Dh * sm[tid * 4 + e];
  }
}

constexpr int kChunk = 64, kTLD = kChunk + 8;
constexpr size_t ssd_smem_bytes(int kt) {
  // C, B [64][dk + 8]; B^T [dk][72]; x^T [128][72] (bf16); four tables of 64 per wave
  return (size_t)(2 * kChunk * (kt * 32 + 8) + kt * 32 * kTLD + 128 * kTLD) * 2 + 4 * 4 * 64 * 4;
}

// A work-group takes one span of one (row, group) and 128 of the group's value columns (heads side by
// side, each padded to whole runs of 32); wave w keeps the state of columns 32 w .. + 31 -- all of one
// head -- in its accumulators (fp32).  Per chunk of 64 tokens, with L the running sum of the logarithms of the
// decays from the chunk's start:
//   y_i = exp(L_i) C_i S + sum_{j <= i} exp(L_i - L_j) dt_j (C_i . B_j) x_j + D x_i
//   S   = exp(L_n) S + sum_j B_j (exp(L_n - L_j) dt_j x_j)^T
// The accumulator layout of S is, in a permuted order of the state dimension that C's fragments follow,
// the B operand of C S; likewise the scores (computed transposed) are the A operand of the product with x.
// fp32 operands (S, weighted scores, weighted x) enter as a high and a low bf16 part.
// STATES: only the span's own contribution to the state and its decay are formed (into ws).
template <int KT, bool STATES>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, KT <= 4 ? 2 : 1))) void ssd_chunk_kernel(const SsdArgs a, const RowSrc<uint16_t> src) {
  constexpr int DK = KT * 32, QLD = DK + 8;
  extern __shared__ __align__(16) unsigned char smem[];
  uint16_t* qs = reinterpret_cast<uint16_t*>(smem);
  uint16_t* ks = qs + kChunk * QLD;
  uint16_t* ktr = ks + kChunk * QLD;
  uint16_t* vt = ktr + DK * kTLD;
  const int tid = threadIdx.x, lane = tid & 63, l32 = lane & 31, lh = lane >> 5;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  float* tl = reinterpret_cast<float*>(vt + 128 * kTLD) + wave * 256;   // L_i in log2 units
  float* td = tl + 64;                                                  // dt_j
  float* te = tl + 128;                                                 // exp(L_i)
  float* tw = tl + 192;                                                 // exp(L_n - L_j) dt_j
  const int span = blockIdx.x % a.n_spans, slice = blockIdx.x / a.n_spans;
  const int g = blockIdx.y;
  const int64_t b = blockIdx.z;
  if (STATES && span == a.n_spans - 1) return;             // nothing starts from the last span's state
  const int col0 = *a.col_ptr, start = a.starts[b];
  const int wcol = slice * 128 + wave * 32;                // this wave's first column in the group
  const int hl = wcol / a.pp;                              // its head in the group
  const bool active = hl < a.hpg;
  const int h = g * a.hpg + (active ? hl : 0);
  const float A2 = -expf(a.A_log[h]) * kLog2e, bias = a.dt_bias[h], Dh = a.D[h];
  const int t_begin = span * a.span, t_end = min((int)a.T, t_begin + a.span);
  const int pcol = wcol % a.pp + l32;                      // this lane's column of the head
  const bool dok = active && pcol < a.P;
  const int64_t ocol = (int64_t)h * a.P + pcol;
  const uint16_t* up = reinterpret_cast<const uint16_t*>(a.u);
  const int64_t inner = (int64_t)a.H * a.P;
  float decay_sum = 0.f;

  f32x16 S[KT];
  {
    const float* init = nullptr;
    if (!STATES) {
      if (a.n_spans > 1) init = a.ws + ((b * a.H + h) * a.n_spans + span) * (int64_t)a.N * a.P;
      else if (col0 > start) init = a.state + (b * a.H + h) * (int64_t)a.N * a.P;
    }
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int r = kt * 32 + 8 * (i >> 2) + 4 * lh + (i & 3);
        S[kt][i] = init && dok && r < a.N ? init[(int64_t)r * a.P + pcol] : 0.f;
      }
  }

  // staging: item = (pair of tokens, eight dimensions)
  constexpr int QI = 32 * (DK / 8) / 256 > 0 ? 32 * (DK / 8) / 256 : 1;   // items per thread of C and of B
  constexpr int VI = 2;                                                   // 32 pairs x 16 runs of x
  u32x4 qr[QI][2], kr[QI][2], vr[VI][2];
  float dt_raw = 0.f;
  const u32x4 zero = u32x4{0, 0, 0, 0};
  const int vc = slice * 128 + (tid & 15) * 8, vh = vc / a.pp, vp = vc % a.pp;   // this thread's run of x columns
  const bool vok = vh < a.hpg && vp < a.P;
  const uint16_t* vsrc = up + (int64_t)(g * a.hpg + (vok ? vh : 0)) * a.P + (vok ? vp : 0);
  auto fetch = [&](int t0) {
#pragma unroll
    for (int c = 0; c < QI; ++c) {
      const int it = c * 256 + tid, pr = it / (DK / 8), ch = it % (DK / 8);
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int t = t0 + 2 * pr + e;
        const bool ok = pr < 32 && ch * 8 < a.N && t < t_end && col0 + t >= start;
        const uint16_t* p = up + (b * a.T + t) * a.u_ld + inner + (int64_t)g * a.N + ch * 8;
        kr[c][e] = ok ? *reinterpret_cast<const u32x4*>(p) : zero;
        if (!STATES) qr[c][e] = ok ? *reinterpret_cast<const u32x4*>(p + (int64_t)a.G * a.N) : zero;
      }
    }
#pragma unroll
    for (int c = 0; c < VI; ++c) {
      const int pr = (c * 256 + tid) / 16;
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int t = t0 + 2 * pr + e;
        vr[c][e] = vok && t < t_end && col0 + t >= start ? *reinterpret_cast<const u32x4*>(vsrc + (b * a.T + t) * a.u_ld) : zero;
      }
    }
    const int t = t0 + lane;
    dt_raw = t < t_end ? src.get(b * a.T + t, a.dt_off + h) : 0.f;
  };
  // two tokens' runs of eight -> eight words (token, next token)
  auto pair_word = [](const u32x4& x, const u32x4& y, int j) -> uint32_t {
    return __builtin_amdgcn_perm(y[j >> 1], x[j >> 1], (j & 1) ? 0x07060302u : 0x05040100u);
  };

  // chunks wholly in front of the sequence change nothing
  int t0 = t_begin;
  if (start > col0) t0 = max(t_begin, t_begin + (start - col0 - t_begin) / kChunk * kChunk);
  if (!STATES && dok)
    for (int t = t_begin + lh; t < min(t0, t_end); t += 2) a.o[(b * a.T + t) * a.o_ld + ocol] = 0.f;
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
    // the decays of this wave's head; tokens outside the sequence neither decay nor add
    const bool real = lane < n && col0 + t0 + lane >= start;
    const float dt = real ? softplus_f32(dt_raw + bias) : 0.f;
    float Ls = A2 * dt;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float v = __shfl_up(Ls, o, 64);
      if (lane >= o) Ls += v;
    }
    const float Ln = __shfl(Ls, 63, 64);
    decay_sum += Ln;
    tl[lane] = Ls;
    td[lane] = dt;
    te[lane] = __builtin_amdgcn_exp2f(Ls);
    tw[lane] = __builtin_amdgcn_exp2f(Ln - Ls) * dt;
    __syncthreads();
    if (t0 + kChunk < t_end) fetch(t0 + kChunk);
    if (!active) continue;                                 // (wave-uniform)
    if constexpr (!STATES) {
      f32x16 O[2];
#pragma unroll
      for (int qt = 0; qt < 2; ++qt)
#pragma unroll
        for (int i = 0; i < 16; ++i) O[qt][i] = 0.f;
      // C S: k index 8 lh + 4 b + e of step s <-> state dimension 32 kt + 16 s + 8 b + 4 lh + e
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
      // the decay in front, and D x
#pragma unroll
      for (int qt = 0; qt < 2; ++qt)
#pragma unroll
        for (int bb = 0; bb < 4; ++bb) {
          const int r0 = qt * 32 + 8 * bb + 4 * lh;
          const f32x4 w = *reinterpret_cast<const f32x4*>(&te[r0]);
          const u32x2 xv = *reinterpret_cast<const u32x2*>(&vt[(wave * 32 + l32) * kTLD + r0]);
          const float xf[4] = {bflo(xv[0]), bfhi(xv[0]), bflo(xv[1]), bfhi(xv[1])};
#pragma unroll
          for (int e = 0; e < 4; ++e) O[qt][4 * bb + e] = O[qt][4 * bb + e] * w[e] + Dh * xf[e];
        }
      // inside the chunk
#pragma unroll
      for (int qt = 0; qt < 2; ++qt) {
        const float Lq = tl[qt * 32 + l32];
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
            const f32x4 Lk = *reinterpret_cast<const f32x4*>(&tl[k0]), dk = *reinterpret_cast<const f32x4*>(&td[k0]);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              const float w = __builtin_amdgcn_exp2f(fminf(Lq - Lk[e], 0.f)) * dk[e];
              st[4 * bb + e] = k0 + e <= qt * 32 + l32 ? st[4 * bb + e] * w : 0.f;
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
            const u32x4 bf = {p0[0], p0[1], p1[0], p1[1]};
            O[qt] = mfma32(ah, bf, O[qt]);
            O[qt] = mfma32(al, bf, O[qt]);
          }
        }
      }
      if (dok)
#pragma unroll
        for (int qt = 0; qt < 2; ++qt)
#pragma unroll
          for (int i = 0; i < 16; ++i) {
            const int r = qt * 32 + 8 * (i >> 2) + 4 * lh + (i & 3);
            if (r < n) a.o[(b * a.T + t0 + r) * a.o_ld + ocol] = O[qt][i];
          }
    }
    // the state behind this chunk
    const float dn = __builtin_amdgcn_exp2f(Ln);
    u32x4 bh[4], bl[4];
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const u32x4 xv = *reinterpret_cast<const u32x4*>(&vt[(wave * 32 + l32) * kTLD + 16 * s + 8 * lh]);
      const f32x4 w0 = *reinterpret_cast<const f32x4*>(&tw[16 * s + 8 * lh]), w1 = *reinterpret_cast<const f32x4*>(&tw[16 * s + 8 * lh + 4]);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float wa = r < 2 ? w0[2 * r] : w1[2 * r - 4], wb = r < 2 ? w0[2 * r + 1] : w1[2 * r - 3];
        uint32_t hi, lo;
        split2(bflo(xv[r]) * wa, bfhi(xv[r]) * wb, hi, lo);
        bh[s][r] = hi;
        bl[s][r] = lo;
      }
    }
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
#pragma unroll
      for (int i = 0; i < 16; ++i) S[kt][i] *= dn;
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        const u32x4 kf = *reinterpret_cast<const u32x4*>(&ktr[(kt * 32 + l32) * kTLD + 16 * s + 8 * lh]);
        S[kt] = mfma32(kf, bh[s], S[kt]);
        S[kt] = mfma32(kf, bl[s], S[kt]);
      }
    }
  }
  if (!dok) return;
  float* dst = nullptr;
  if (STATES) dst = a.ws + ((b * a.H + h) * a.n_spans + span) * (int64_t)a.N * a.P;
  else if (span == a.n_spans - 1) dst = a.state + (b * a.H + h) * (int64_t)a.N * a.P;
  if (dst)
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int r = kt * 32 + 8 * (i >> 2) + 4 * lh + (i & 3);
        if (r < a.N) dst[(int64_t)r * a.P + pcol] = S[kt][i];
      }
  if (STATES && pcol == 0 && lh == 0)
    a.ws[a.B * a.H * a.n_spans * (int64_t)a.N * a.P + (b * a.H + h) * a.n_spans + span] = __builtin_amdgcn_exp2f(decay_sum);
}

// the spans' own contributions -> the state each span starts from, in place
__global__ __launch_bounds__(256) void ssd_scan_kernel(const SsdArgs a) {
  const int64_t n = (int64_t)a.N * a.P, i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  const int h = blockIdx.y;
  const int64_t b = blockIdx.z;
  if (i >= n) return;
  float cur = *a.col_ptr > a.starts[b] ? a.state[(b * a.H + h) * n + i] : 0.f;
  float* p = a.ws + (b * a.H + h) * a.n_spans * n + i;
  const float* dec = a.ws + a.B * a.H * a.n_spans * n + (b * a.H + h) * a.n_spans;
  for (int s = 0; s < a.n_spans; ++s) {
    const bool more = s + 1 < a.n_spans;
    const float u = more ? p[s * n] : 0.f, d = more ? dec[s] : 0.f;
    p[s * n] = cur;
    cur = d * cur + u;
  }
}

template <int KT>
int launch_chunk(hipStream_t st, const SsdArgs& a, const RowSrc<uint16_t>& src) {
  static std::once_flag once;
  static hipError_t e = hipSuccess;
  constexpr size_t kSmem = ssd_smem_bytes(KT);
  std::call_once(once, [] {
    e = hipFuncSetAttribute(reinterpret_cast<const void*>(&ssd_chunk_kernel<KT, false>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kSmem);
    if (e == hipSuccess)
      e = hipFuncSetAttribute(reinterpret_cast<const void*>(&ssd_chunk_kernel<KT, true>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kSmem);
  });
  if (e != hipSuccess) {
    tnx_set_error("ssd: cannot raise the dynamic LDS limit: %s", hipGetErrorString(e));
    return TNX_ELAUNCH;
  }
  const dim3 grid((unsigned)(a.n_spans * a.slices), (unsigned)a.G, (unsigned)a.B);
  if (a.n_spans > 1) {
    hipLaunchKernelGGL((ssd_chunk_kernel<KT, true>), grid, dim3(256), kSmem, st, a, src);
    hipLaunchKernelGGL(ssd_scan_kernel, dim3((unsigned)cdiv((int64_t)a.N * a.P, 256), (unsigned)a.H, (unsigned)a.B), dim3(256), 0, st, a);
  }
  hipLaunchKernelGGL((ssd_chunk_kernel<KT, false>), grid, dim3(256), kSmem, st, a, src);
  TNX_CHECK_LAUNCH("ssd_chunk");
  return TNX_OK;
}

int padded_cols(int P) { return (P + 31) / 32 * 32; }
int64_t slices_of(int hpg, int P) { return cdiv((int64_t)hpg * padded_cols(P), 128); }
// work-groups of a prompt pass that fill the device; shorter spans cost state traffic
int span_tokens(int64_t B, int64_t T, int H, int G, int P) {
  const int64_t per = B * G * slices_of(H / G, P);
  int64_t spans = per >= 256 ? 1 : cdiv(512, per);
  int64_t span = cdiv(cdiv(T, spans), kChunk) * kChunk;
  if (span < 2 * kChunk) span = 2 * kChunk;
  return (int)span;
}

template <typename T>
int conv_launch(hipStream_t st, const tnx_short_conv_desc* d, const ConvArgs& a) {
  const RowSrc<T> src{(const T*)d->y.y, d->y.ws, d->y.split_k, d->y.plane, d->y.ld};
  const bool vec = a.C % 8 == 0 && a.off % 8 == 0 && d->y.ld % 8 == 0 && d->y.plane % 8 == 0 && a.out_ld % 8 == 0 && a.taps >= 2 && a.taps <= 4;
  if (vec) {
    int run = kConvRun;
    while (run > 1 && a.B * cdiv(a.T, run) * (a.C / 8) < 131072) run /= 2;
    const int64_t items = a.B * cdiv(a.T, run) * (a.C / 8);
    const dim3 grid((unsigned)cdiv(items, 256));
    if (a.taps == 2) hipLaunchKernelGGL((short_conv_vec_kernel<2, T>), grid, dim3(256), 0, st, a, src, run);
    else if (a.taps == 3) hipLaunchKernelGGL((short_conv_vec_kernel<3, T>), grid, dim3(256), 0, st, a, src, run);
    else hipLaunchKernelGGL((short_conv_vec_kernel<4, T>), grid, dim3(256), 0, st, a, src, run);
  } else {
    const int64_t rows = a.B * a.T;
    hipLaunchKernelGGL(short_conv_kernel<T>, dim3((unsigned)cdiv(a.C, 256), (unsigned)(rows < 32768 ? rows : 32768), (unsigned)cdiv(rows, 32768)),
                       dim3(256), 0, st, a, src);
  }
  TNX_CHECK_LAUNCH("short_conv");
  return TNX_OK;
}

}  // namespace

extern "C" int tnx_short_conv(void* stream, const tnx_short_conv_desc* d) {
  TNX_REQUIRE(d, "short_conv: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->T > 0 && d->C > 0 && d->taps > 0 && d->taps <= 4096 && d->slots >= d->taps - 1 && d->slots > 0, "short_conv: bad shape");
  TNX_REQUIRE(src_given(d->y) && d->w && d->bias && d->ring && d->starts && d->col_ptr && d->out && d->out_ld >= d->C, "short_conv: null pointer or short rows");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "short_conv: bad dtype %d", d->dtype);
  TNX_REQUIRE(d->B * d->T < (int64_t)1 << 30, "short_conv: too many rows");
  ConvArgs a;
  a.B = d->B; a.T = d->T; a.C = d->C; a.off = d->off; a.out_ld = d->out_ld; a.taps = d->taps; a.slots = d->slots; a.w = d->w;
  a.bias = d->bias; a.ring = d->ring; a.starts = d->starts; a.col_ptr = d->col_ptr; a.out = d->out;
  return d->dtype == TNX_BF16 ? conv_launch<uint16_t>(as_stream(stream), d, a) : conv_launch<float>(as_stream(stream), d, a);
}

extern "C" int tnx_ring_write(void* stream, int dtype, const tnx_rows_src* y, int64_t off, int64_t B, int64_t T, int64_t C, int slots,
                              const int32_t* col_ptr, int64_t t0, void* ring) {
  TNX_REQUIRE(y && src_given(*y) && col_ptr && ring, "ring_write: null pointer");
  TNX_REQUIRE(B > 0 && B <= 65535 && T > 0 && C > 0 && slots > 0 && slots <= 65535 && off >= 0 && t0 >= 0, "ring_write: bad shape");
  TNX_REQUIRE(dtype == TNX_BF16 || dtype == TNX_F32, "ring_write: bad dtype %d", dtype);
  const dim3 grid((unsigned)cdiv(C, 256), (unsigned)(T < slots ? T : slots), (unsigned)B);
  if (dtype == TNX_BF16) {
    const RowSrc<uint16_t> s{(const uint16_t*)y->y, y->ws, y->split_k, y->plane, y->ld};
    hipLaunchKernelGGL(ring_write_kernel<uint16_t>, grid, dim3(256), 0, as_stream(stream), T, C, off, slots, col_ptr, t0, s, (uint16_t*)ring);
  } else {
    const RowSrc<float> s{(const float*)y->y, y->ws, y->split_k, y->plane, y->ld};
    hipLaunchKernelGGL(ring_write_kernel<float>, grid, dim3(256), 0, as_stream(stream), T, C, off, slots, col_ptr, t0, s, (float*)ring);
  }
  TNX_CHECK_LAUNCH("ring_write");
  return TNX_OK;
}

extern "C" size_t tnx_ssd_ws_bytes(int64_t B, int64_t T, int H, int G, int N, int P) {
  if (T <= 1 || B <= 0 || H <= 0 || G <= 0 || H % G) return 0;
  const int64_t spans = cdiv(T, span_tokens(B, T, H, G, P));
  return spans > 1 ? (size_t)(B * H * spans) * ((size_t)N * (size_t)P + 1) * 4 : 0;
}

extern "C" int tnx_ssd_step_ok(int N, int P) { return P % 4 == 0 && P <= 1024 && P + 2 * N <= 8192; }

extern "C" int tnx_ssd(void* stream, const tnx_ssd_desc* d) {
  TNX_REQUIRE(d, "ssd: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->T > 0 && d->H > 0 && d->G > 0 && d->H % d->G == 0 && d->N > 0 && d->P > 0, "ssd: bad shape");
  TNX_REQUIRE(d->A_log && d->dt_bias && d->D && d->starts && d->col_ptr && d->state && d->o && src_given(d->y), "ssd: null pointer");
  TNX_REQUIRE(d->o_ld >= (int64_t)d->H * d->P && d->N <= 8192, "ssd: short output rows or a state size above 8192");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "ssd: bad dtype %d", d->dtype);
  TNX_REQUIRE(d->B <= 65535 && d->H <= 65535, "ssd: too many rows or heads");
  SsdArgs a;
  memset(&a, 0, sizeof(a));
  a.B = d->B; a.T = d->T; a.H = d->H; a.G = d->G; a.N = d->N; a.P = d->P; a.hpg = d->H / d->G; a.A_log = d->A_log; a.dt_bias = d->dt_bias;
  a.D = d->D; a.starts = d->starts; a.col_ptr = d->col_ptr; a.dt_off = d->dt_off; a.o_ld = d->o_ld; a.state = d->state; a.o = d->o;
  a.u = d->u; a.u_ld = d->u_ld;
  hipStream_t st = as_stream(stream);
  const bool bf = d->dtype == TNX_BF16;
  const RowSrc<uint16_t> s16{(const uint16_t*)d->y.y, d->y.ws, d->y.split_k, d->y.plane, d->y.ld};
  const RowSrc<float> s32{(const float*)d->y.y, d->y.ws, d->y.split_k, d->y.plane, d->y.ld};
  const dim3 per((unsigned)d->H, (unsigned)d->B);
  if (!d->u) {   // one token, the convolution inside
    TNX_REQUIRE(d->T == 1 && tnx_ssd_step_ok(d->N, d->P), "ssd: this shape needs convolved rows");
    TNX_REQUIRE(d->conv_w && d->conv_b && d->ring && d->taps > 0 && d->slots >= d->taps, "ssd: the step needs the convolution and a ring of at least its taps");
    a.c_off = d->c_off; a.taps = d->taps; a.slots = d->slots; a.conv_w = d->conv_w; a.conv_b = d->conv_b; a.ring = d->ring;
    const size_t lds = (size_t)((d->P + 2 * d->N + 3) / 4 * 4 + 1024) * 4;
    if (bf) hipLaunchKernelGGL(ssd_step_kernel<uint16_t>, per, dim3(256), lds, st, a, s16);
    else hipLaunchKernelGGL(ssd_step_kernel<float>, per, dim3(256), lds, st, a, s32);
    TNX_CHECK_LAUNCH("ssd_step");
    return TNX_OK;
  }
  TNX_REQUIRE(d->u_ld >= (int64_t)d->H * d->P + 2 * (int64_t)d->G * d->N, "ssd: short rows");
  if (bf && d->T > 1 && d->N % 8 == 0 && d->N <= 256 && d->P % 8 == 0 && d->u_ld % 8 == 0 && d->T < (1 << 30)) {
    a.pp = padded_cols(d->P);
    a.slices = (int)slices_of(a.hpg, d->P);
    a.span = span_tokens(d->B, d->T, d->H, d->G, d->P);
    a.n_spans = (int)cdiv(d->T, a.span);
    a.ws = d->ws;
    TNX_REQUIRE(d->G <= 65535, "ssd: too many groups");
    TNX_REQUIRE(a.n_spans == 1 || d->ws, "ssd: a long prompt needs the workspace of tnx_ssd_ws_bytes");
    if (d->N <= 32) return launch_chunk<1>(st, a, s16);
    if (d->N <= 64) return launch_chunk<2>(st, a, s16);
    if (d->N <= 128) return launch_chunk<4>(st, a, s16);
    return launch_chunk<8>(st, a, s16);
  }
  const size_t lds = (size_t)2 * d->N * 4;
  if (bf) hipLaunchKernelGGL(ssd_any_kernel<uint16_t>, per, dim3(256), lds, st, a, s16);
  else hipLaunchKernelGGL(ssd_any_kernel<float>, per, dim3(256), lds, st, a, s32);
  TNX_CHECK_LAUNCH("ssd_any");
  return TNX_OK;
}
