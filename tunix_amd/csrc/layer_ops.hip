// Small operations of decoders with dense weights whose layers are averaged over depth: the residual step with
// centred norms, a factor, an extra row and the average over earlier layers' results; query and key norms over a whole
// projection with the cache write; PolyNorm; the choice of experts by corrected scores.  All of it in 32-bit; matrix
// operands leave in the model's dtype.
#include <string.h>

#include <type_traits>

#include "decoder.h"

namespace {

template <typename T>
RowSrc<T> row_src(const tnx_rows_src& s) {
  return RowSrc<T>{reinterpret_cast<const T*>(s.y), s.ws, s.split_k < 1 ? 1 : s.split_k, s.plane, s.ld};
}
__device__ __forceinline__ void load8f(const float* p, float (&f)[8]) {
  const f32x4 u = *reinterpret_cast<const f32x4*>(p), v = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    f[j] = u[j];
    f[4 + j] = v[j];
  }
}
__device__ __forceinline__ float block_total(float v, float* red) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
  for (int w = 0; w < (int)(blockDim.x >> 6); ++w) s += red[w];
  return s;
}

// ---- residual step ------------------------------------------------------------------------------
struct StepArgs {
  int64_t D;
  float eps, w_offset, mult;
  int mode;                // 0: nothing arrives, 1: x + mult norm(y) . w_post
  const float* w_post;
  const float* x;
  float* x_out;            // null: x stays
  const float* route_w;
  int route_k;
  const float* extra_w;
  bool has_extra;
  float* hist;
  int64_t hist_plane;
  int hist_n, hist_store;
  const float* hist_w;
  const float* w_next;
  void* out;
  int64_t out_ld;
  int out_frag;
};

// A row per work-group, eight elements per thread and run; everything the row needs is requested before the first sum,
// the earlier results included.
template <int NT, int MAXC, bool ROUTES, bool CENTER, typename T>   // NT threads, MAXC runs of eight per thread
__global__ __launch_bounds__(NT) void layer_step_kernel(const StepArgs a, const RowSrc<T> y, const RowSrc<T> extra) {
  constexpr int NW = NT / 64;
  __shared__ float red[2][NW][2];
  const int64_t row = blockIdx.x;
  const int nch = (int)(a.D / 8), tid = threadIdx.x, wave = tid >> 6;
  auto column = [&](int c) { return (int64_t)min(c * NT + tid, nch - 1) * 8; };
  auto elements = [&](int w) {   // of a wave
    int n = 0;
#pragma unroll
    for (int c = 0; c < MAXC; ++c) n += max(0, min(64, nch - c * NT - w * 64));
    return (float)(8 * n);
  };
  float h[MAXC][8], xo[MAXC][8], wp[MAXC][8], wn[MAXC][8], past[MAXC][8];
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int64_t col = column(c);
    load8f(a.x + row * a.D + col, xo[c]);
    if (a.mode == 1) {
      load8f(a.w_post + col, wp[c]);
      if constexpr (ROUTES) {
#pragma unroll
        for (int j = 0; j < 8; ++j) h[c][j] = 0.f;
#pragma unroll 4
        for (int k = 0; k < a.route_k; ++k) {
          const float w = a.route_w[row * a.route_k + k];
          float f[8];
          get8(RowSrc<T>{y.y, nullptr, 1, 0, y.ld}, row * a.route_k + k, col, f);
#pragma unroll
          for (int j = 0; j < 8; ++j) h[c][j] += w * f[j];
        }
      } else {
        get8(y, row, col, h[c]);
      }
      if (a.has_extra) {
        const float w = a.extra_w ? a.extra_w[row] : 1.f;
        float f[8];
        get8(extra, row, col, f);
#pragma unroll
        for (int j = 0; j < 8; ++j) h[c][j] += w * f[j];
      }
    }
    if (a.w_next) load8f(a.w_next + col, wn[c]);
#pragma unroll
    for (int j = 0; j < 8; ++j) past[c][j] = 0.f;
    if (a.hist)
#pragma unroll 4
      for (int k = 0; k < a.hist_n; ++k) {
        float f[8];
        load8f(a.hist + k * a.hist_plane + row * a.D + col, f);
        const float w = a.hist_w[k];
#pragma unroll
        for (int j = 0; j < 8; ++j) past[c][j] += w * f[j];
      }
  }
  // mean (0 without CENTER) and 1 / sqrt(variance + eps): every wave about its own mean, then merged
  auto moments = [&](const float (&v)[MAXC][8], float (*rd)[2], float& mean, float& r) {
    float s = 0.f, q = 0.f, own = 0.f;
    if constexpr (CENTER) {
#pragma unroll
      for (int c = 0; c < MAXC; ++c)
        if (c * NT + tid < nch)
#pragma unroll
          for (int j = 0; j < 8; ++j) s += v[c][j];
      s = wave_sum(s);
      own = s / fmaxf(elements(wave), 1.f);
    }
#pragma unroll
    for (int c = 0; c < MAXC; ++c)
      if (c * NT + tid < nch)
#pragma unroll
        for (int j = 0; j < 8; ++j) q += (v[c][j] - own) * (v[c][j] - own);
    q = wave_sum(q);
    if ((tid & 63) == 0) {
      rd[wave][0] = s;
      rd[wave][1] = q;
    }
    __syncthreads();
    float sum = 0.f, m2 = 0.f;
    mean = 0.f;
    if constexpr (CENTER) {
#pragma unroll
      for (int w = 0; w < NW; ++w) sum += rd[w][0];
      mean = sum / (float)a.D;
    }
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      m2 += rd[w][1];
      if constexpr (CENTER) {
        const float n = elements(w), d = rd[w][0] / fmaxf(n, 1.f) - mean;
        m2 += n * d * d;
      }
    }
    r = 1.0f / sqrtf(m2 / (float)a.D + a.eps);
  };
  float mean, r;
  if (a.mode == 1) moments(h, red[0], mean, r);
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const bool mine = c * NT + tid < nch;
    const int64_t at = row * a.D + column(c);
#pragma unroll
    for (int j = 0; j < 8; ++j)
      h[c][j] = a.mode == 1 ? xo[c][j] + a.mult * ((h[c][j] - mean) * r * (a.w_offset + wp[c][j])) : xo[c][j];
    if (a.hist) {
      if (a.hist_store && mine) put8(a.hist + a.hist_n * a.hist_plane + at, h[c]);
      const float w = a.hist_w[a.hist_n];
#pragma unroll
      for (int j = 0; j < 8; ++j) h[c][j] = past[c][j] + w * h[c][j];
    }
    if (a.x_out && mine) put8(a.x_out + at, h[c]);
  }
  if (a.w_next) moments(h, red[1], mean, r);
  T* out = reinterpret_cast<T*>(a.out);
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    if (c * NT + tid >= nch) continue;
    const int64_t col = column(c);
    if (a.w_next)
#pragma unroll
      for (int j = 0; j < 8; ++j) h[c][j] = (h[c][j] - mean) * r * (a.w_offset + wn[c][j]);
    put8(out + (a.out_frag ? frag_index(row, col, a.out_ld) : row * a.out_ld + col), h[c]);
  }
}

// any D that fits LDS
template <bool CENTER, typename T>
__global__ __launch_bounds__(256) void layer_step_any_kernel(const StepArgs a, const RowSrc<T> y, const RowSrc<T> extra) {
  extern __shared__ __align__(16) float hrow[];
  __shared__ float red[4];
  const int64_t row = blockIdx.x;
  float mean = 0.f, r = 1.f;
  auto moments = [&]() {   // (a thread reads the elements it has written)
    float s = 0.f;
    mean = 0.f;
    if constexpr (CENTER) {
      for (int64_t i = threadIdx.x; i < a.D; i += 256) s += hrow[i];
      mean = block_total(s, red) / (float)a.D;
      s = 0.f;
    }
    for (int64_t i = threadIdx.x; i < a.D; i += 256) s += (hrow[i] - mean) * (hrow[i] - mean);
    r = 1.0f / sqrtf(block_total(s, red) / (float)a.D + a.eps);
  };
  if (a.mode == 1) {
    for (int64_t i = threadIdx.x; i < a.D; i += 256) {
      float v = 0.f;
      if (a.route_w)
        for (int k = 0; k < a.route_k; ++k) v += a.route_w[row * a.route_k + k] * y.get(row * a.route_k + k, i);
      else v = y.get(row, i);
      if (a.has_extra) v += (a.extra_w ? a.extra_w[row] : 1.f) * extra.get(row, i);
      hrow[i] = v;
    }
    moments();
  }
  for (int64_t i = threadIdx.x; i < a.D; i += 256) {
    const int64_t at = row * a.D + i;
    float v = a.x[at];
    if (a.mode == 1) v += a.mult * ((hrow[i] - mean) * r * (a.w_offset + a.w_post[i]));
    if (a.hist) {
      float past = 0.f;
      for (int k = 0; k < a.hist_n; ++k) past += a.hist_w[k] * a.hist[k * a.hist_plane + at];
      if (a.hist_store) a.hist[a.hist_n * a.hist_plane + at] = v;
      v = past + a.hist_w[a.hist_n] * v;
    }
    if (a.x_out) a.x_out[at] = v;
    hrow[i] = v;
  }
  if (a.w_next) moments();
  T* out = reinterpret_cast<T*>(a.out);
  for (int64_t i = threadIdx.x; i < a.D; i += 256) {
    const float v = a.w_next ? (hrow[i] - mean) * r * (a.w_offset + a.w_next[i]) : hrow[i];
    st_elem(out, a.out_frag ? frag_index(row, i, a.out_ld) : row * a.out_ld + i, v);
  }
}

template <bool CENTER, typename T>
int launch_step(hipStream_t st, int64_t M, const StepArgs& a, const RowSrc<T>& y, const RowSrc<T>& extra) {
  const dim3 grid((unsigned)M);
  const bool vec = a.D % 8 == 0 && a.out_ld % 8 == 0 && a.hist_plane % 8 == 0 && (a.mode == 0 || (y.ld % 8 == 0 && y.plane % 8 == 0)) &&
                   (!a.has_extra || (extra.ld % 8 == 0 && extra.plane % 8 == 0));
  if (!vec) {
    TNX_REQUIRE(a.D <= 14336, "residual_norm: D=%lld needs runs of eight", (long long)a.D);
    hipLaunchKernelGGL((layer_step_any_kernel<CENTER, T>), grid, dim3(256), (size_t)a.D * 4, st, a, y, extra);
    TNX_CHECK_LAUNCH("residual_norm");
    return TNX_OK;
  }
  auto launch = [&](auto routes) {
    constexpr bool R = decltype(routes)::value;
    if (a.D <= 2048) hipLaunchKernelGGL((layer_step_kernel<256, 1, R, CENTER, T>), grid, dim3(256), 0, st, a, y, extra);
    else if (a.D <= 4096) hipLaunchKernelGGL((layer_step_kernel<512, 1, R, CENTER, T>), grid, dim3(512), 0, st, a, y, extra);
    else if (a.D <= 8192) hipLaunchKernelGGL((layer_step_kernel<1024, 1, R, CENTER, T>), grid, dim3(1024), 0, st, a, y, extra);
    else hipLaunchKernelGGL((layer_step_kernel<1024, 2, R, CENTER, T>), grid, dim3(1024), 0, st, a, y, extra);
  };
  if (a.route_w) launch(std::true_type{});
  else launch(std::false_type{});
  TNX_CHECK_LAUNCH("residual_norm");
  return TNX_OK;
}

// ---- norms over whole projections, cache write ------------------------------------------------------
struct RowNormArgs {
  int64_t T, S;
  int H, G, dk, dv, dkp, dvp;
  float eps;
  const float* w_q;
  const float* w_k;
  int64_t k_off, v_off;
  const int32_t* col_ptr;
};
// An item is eight dimensions of one padded head: queries, then (kc not null) keys and values.
template <int NT, int MAXC, typename T>
__global__ __launch_bounds__(NT) void rownorm_kv_kernel(const RowNormArgs a, const RowSrc<T> src, T* q_out, T* kc, T* vc) {
  __shared__ float red[NT / 64][2];
  const int64_t row = blockIdx.x, b = row / a.T, t = row % a.T;
  const int tid = threadIdx.x, kch = a.dkp / 8, vch = a.dvp / 8;
  const int nq = a.H * kch, nk = kc ? nq + a.G * kch : nq, n = kc ? nk + a.G * vch : nq;
  const int slot = *a.col_ptr + (int)t;
  if (slot >= a.S) return;                                    // (uniform; the host sizes the cache)
  float v[MAXC][8], w[MAXC][8];
  int kind[MAXC];                                             // 0 q, 1 k, 2 v, 3 padding, 4 none
  T* dst[MAXC];
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int it = c * NT + tid;
    kind[c] = it < nq ? 0 : it < nk ? 1 : it < n ? 2 : 4;
    dst[c] = nullptr;
#pragma unroll
    for (int j = 0; j < 8; ++j) v[c][j] = w[c][j] = 0.f;
    if (kind[c] == 4) continue;
    const int i = kind[c] == 0 ? it : kind[c] == 1 ? it - nq : it - nk, ch = kind[c] == 2 ? vch : kch, dim = kind[c] == 2 ? a.dv : a.dk;
    const int hd = i / ch, d = i % ch * 8;
    dst[c] = (kind[c] == 0 ? q_out + (row * a.H + hd) * a.dkp : kind[c] == 1 ? kc + ((b * a.G + hd) * a.S + slot) * a.dkp
                                                                            : vc + ((b * a.G + hd) * a.S + slot) * a.dvp) + d;
    if (d >= dim) {
      kind[c] = 3;
      continue;
    }
    const int64_t at = (int64_t)hd * dim + d;
    get8(src, row, (kind[c] == 0 ? 0 : kind[c] == 1 ? a.k_off : a.v_off) + at, v[c]);
    if (kind[c] < 2) load8f((kind[c] == 0 ? a.w_q : a.w_k) + at, w[c]);
  }
  float sq = 0.f, sk = 0.f;
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) s += v[c][j] * v[c][j];
    if (kind[c] == 0) sq += s;
    if (kind[c] == 1) sk += s;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((tid & 63) == 0) {
    red[tid >> 6][0] = sq;
    red[tid >> 6][1] = sk;
  }
  __syncthreads();
  sq = sk = 0.f;
#pragma unroll
  for (int i = 0; i < NT / 64; ++i) {
    sq += red[i][0];
    sk += red[i][1];
  }
  const float rq = 1.0f / sqrtf(sq / (float)(a.H * a.dk) + a.eps), rk = 1.0f / sqrtf(sk / (float)(a.G * a.dk) + a.eps);
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    if (kind[c] == 4) continue;
    const float r = kind[c] == 0 ? rq : rk;
    if (kind[c] < 2)
#pragma unroll
      for (int j = 0; j < 8; ++j) v[c][j] = v[c][j] * r * w[c][j];
    put8(dst[c], v[c]);
  }
}
// any sizes
template <typename T>
__global__ __launch_bounds__(256) void rownorm_kv_any_kernel(const RowNormArgs a, const RowSrc<T> src, T* q_out, T* kc, T* vc) {
  __shared__ float red[4];
  const int64_t row = blockIdx.x, b = row / a.T, t = row % a.T;
  const int slot = *a.col_ptr + (int)t;
  if (slot >= a.S) return;                                    // (uniform)
  auto norm = [&](int64_t off, int n) {
    float s = 0.f;
    for (int i = threadIdx.x; i < n; i += 256) {
      const float v = src.get(row, off + i);
      s += v * v;
    }
    return 1.0f / sqrtf(block_total(s, red) / (float)n + a.eps);
  };
  const float rq = norm(0, a.H * a.dk);
  for (int it = threadIdx.x; it < a.H * a.dkp; it += 256) {
    const int64_t h = it / a.dkp, i = it % a.dkp;
    st_elem(q_out, (row * a.H + h) * a.dkp + i, i < a.dk ? src.get(row, h * a.dk + i) * rq * a.w_q[h * a.dk + i] : 0.f);
  }
  if (!kc) return;
  const float rk = norm(a.k_off, a.G * a.dk);
  for (int it = threadIdx.x; it < a.G * a.dkp; it += 256) {
    const int64_t g = it / a.dkp, i = it % a.dkp;
    st_elem(kc, ((b * a.G + g) * a.S + slot) * a.dkp + i, i < a.dk ? src.get(row, a.k_off + g * a.dk + i) * rk * a.w_k[g * a.dk + i] : 0.f);
  }
  for (int it = threadIdx.x; it < a.G * a.dvp; it += 256) {
    const int64_t g = it / a.dvp, i = it % a.dvp;
    st_elem(vc, ((b * a.G + g) * a.S + slot) * a.dvp + i, i < a.dv ? src.get(row, a.v_off + g * a.dv + i) : 0.f);
  }
}
template <typename T>
int launch_rownorm_kv(hipStream_t st, int64_t M, const RowNormArgs& a, const RowSrc<T>& src, T* q, T* k, T* v) {
  const dim3 grid((unsigned)M);
  const int64_t items = (int64_t)a.H * a.dkp / 8 + (k ? (int64_t)a.G * (a.dkp + a.dvp) / 8 : 0);
  const bool vec = (a.dk | a.dkp) % 8 == 0 && (!k || ((a.dv | a.dvp) % 8 == 0 && (a.k_off | a.v_off) % 8 == 0)) && src.ld % 8 == 0 && src.plane % 8 == 0;
  if (vec && items <= 256) hipLaunchKernelGGL((rownorm_kv_kernel<256, 1, T>), grid, dim3(256), 0, st, a, src, q, k, v);
  else if (vec && items <= 512) hipLaunchKernelGGL((rownorm_kv_kernel<512, 1, T>), grid, dim3(512), 0, st, a, src, q, k, v);
  else if (vec && items <= 1024) hipLaunchKernelGGL((rownorm_kv_kernel<512, 2, T>), grid, dim3(512), 0, st, a, src, q, k, v);
  else if (vec && items <= 4096) hipLaunchKernelGGL((rownorm_kv_kernel<1024, 4, T>), grid, dim3(1024), 0, st, a, src, q, k, v);
  else hipLaunchKernelGGL((rownorm_kv_any_kernel<T>), grid, dim3(256), 0, st, a, src, q, k, v);
  TNX_CHECK_LAUNCH("rownorm_kvwrite");
  return TNX_OK;
}

// ---- PolyNorm -------------------------------------------------------------------------------------
template <int NT, int MAXC, typename T>
__global__ __launch_bounds__(NT) void poly_norm_kernel(const RowSrc<T> src, int64_t F, const float* coef, float eps, T* out, int64_t out_ld, int out_frag) {
  __shared__ float red[NT / 64][3];
  const int64_t row = blockIdx.x;
  const int nch = (int)(F / 8), tid = threadIdx.x;
  float z[MAXC][8], s[3] = {0.f, 0.f, 0.f};
  const float ca = coef[0], cb = coef[1], cc = coef[2], ce = coef[3];
#pragma unroll
  for (int c = 0; c < MAXC; ++c) get8(src, row, (int64_t)min(c * NT + tid, nch - 1) * 8, z[c]);
#pragma unroll
  for (int c = 0; c < MAXC; ++c)
    if (c * NT + tid < nch)
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float q = z[c][j] * z[c][j];
        s[0] += q;
        s[1] += q * q;
        s[2] += q * q * q;
      }
#pragma unroll
  for (int k = 0; k < 3; ++k) {
    s[k] = wave_sum(s[k]);
    if ((tid & 63) == 0) red[tid >> 6][k] = s[k];
  }
  __syncthreads();
  float r[3];
#pragma unroll
  for (int k = 0; k < 3; ++k) {
    float t = 0.f;
#pragma unroll
    for (int w = 0; w < NT / 64; ++w) t += red[w][k];
    r[k] = 1.0f / sqrtf(t / (float)F + eps);
  }
  r[0] *= ca;
  r[1] *= cb;
  r[2] *= cc;
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    if (c * NT + tid >= nch) continue;
    const int64_t col = (int64_t)(c * NT + tid) * 8;
#pragma unroll
    for (int j = 0; j < 8; ++j) z[c][j] = z[c][j] * (r[0] + z[c][j] * (r[1] + z[c][j] * r[2])) + ce;
    put8(out + (out_frag ? frag_index(row, col, out_ld) : row * out_ld + col), z[c]);
  }
}
template <typename T>
__global__ __launch_bounds__(256) void poly_norm_any_kernel(const RowSrc<T> src, int64_t F, const float* coef, float eps, T* out, int64_t out_ld, int out_frag) {
  __shared__ float red[4];
  const int64_t row = blockIdx.x;
  float s[3] = {0.f, 0.f, 0.f}, r[3];
  for (int64_t i = threadIdx.x; i < F; i += 256) {
    const float z = src.get(row, i), q = z * z;
    s[0] += q;
    s[1] += q * q;
    s[2] += q * q * q;
  }
#pragma unroll
  for (int k = 0; k < 3; ++k) r[k] = coef[k] / sqrtf(block_total(s[k], red) / (float)F + eps);
  for (int64_t i = threadIdx.x; i < F; i += 256) {
    const float z = src.get(row, i);
    st_elem(out, out_frag ? frag_index(row, i, out_ld) : row * out_ld + i, z * (r[0] + z * (r[1] + z * r[2])) + coef[3]);
  }
}
template <typename T>
int launch_poly(hipStream_t st, int64_t M, const RowSrc<T>& src, int64_t F, const float* coef, float eps, T* out, int64_t out_ld, int out_frag) {
  const dim3 grid((unsigned)M);
  const bool vec = F % 8 == 0 && F <= 32768 && src.ld % 8 == 0 && src.plane % 8 == 0 && out_ld % 8 == 0;
  if (!vec) hipLaunchKernelGGL((poly_norm_any_kernel<T>), grid, dim3(256), 0, st, src, F, coef, eps, out, out_ld, out_frag);
  else if (M >= 1024 && F > 2048 && F <= 16384) {   // many rows fill the device: fewer waves meet per row
    if (F <= 4096) hipLaunchKernelGGL((poly_norm_kernel<256, 2, T>), grid, dim3(256), 0, st, src, F, coef, eps, out, out_ld, out_frag);
    else if (F <= 8192) hipLaunchKernelGGL((poly_norm_kernel<256, 4, T>), grid, dim3(256), 0, st, src, F, coef, eps, out, out_ld, out_frag);
    else hipLaunchKernelGGL((poly_norm_kernel<512, 4, T>), grid, dim3(512), 0, st, src, F, coef, eps, out, out_ld, out_frag);
  } else if (F <= 2048) hipLaunchKernelGGL((poly_norm_kernel<256, 1, T>), grid, dim3(256), 0, st, src, F, coef, eps, out, out_ld, out_frag);
  else if (F <= 4096) hipLaunchKernelGGL((poly_norm_kernel<512, 1, T>), grid, dim3(512), 0, st, src, F, coef, eps, out, out_ld, out_frag);
  else if (F <= 8192) hipLaunchKernelGGL((poly_norm_kernel<1024, 1, T>), grid, dim3(1024), 0, st, src, F, coef, eps, out, out_ld, out_frag);
  else if (F <= 16384) hipLaunchKernelGGL((poly_norm_kernel<1024, 2, T>), grid, dim3(1024), 0, st, src, F, coef, eps, out, out_ld, out_frag);
  else hipLaunchKernelGGL((poly_norm_kernel<1024, 4, T>), grid, dim3(1024), 0, st, src, F, coef, eps, out, out_ld, out_frag);
  TNX_CHECK_LAUNCH("poly_norm");
  return TNX_OK;
}

// ---- choice of experts by corrected scores ------------------------------------------------------------
// One wave per token: softmax over all logits, the k largest scores + correction (first among equals).  Whatever the
// logits hold, k distinct experts are found; a row with a NaN leaves NaN weights.
constexpr int kRankedExperts = 256;   // up to here every expert counts the ones ahead of it
__global__ __launch_bounds__(64) void route_scores_kernel(const RowSrc<float> src, int E, int k, const float* correction, float scale, int64_t gate_off,
                                                          int ld, float* topk_w, int32_t* topk_id, float* gate_w) {
  extern __shared__ __align__(16) float lds[];   // choice scores [E rounded up to 4], scores [E], chosen scores [k]
  float *choice = lds, *score = lds + (E + 3) / 4 * 4, *sel = score + E;
  const int64_t m = blockIdx.x;
  const int lane = threadIdx.x;
  const float ninf = -__builtin_inff();
  float top = -3.0e38f;
  bool bad = false;
  for (int e = lane; e < E; e += 64) {
    const float v = src.get(m, e);
    bad |= v != v;
    const float z = v == v ? fminf(fmaxf(v, -3.0e38f), 3.0e38f) : -3.0e38f;
    score[e] = z;
    top = fmaxf(top, z);
  }
  if ((gate_w || ld > k) && lane == 0) {
    const float g = sigmoid_f32(src.get(m, gate_off));
    if (gate_w) gate_w[m] = g;
    for (int j = k; j < ld; ++j) {
      topk_w[m * ld + j] = g;
      topk_id[m * ld + j] = E + j - k;
    }
  }
  bad = __any(bad);
  top = wave_max(top);
  float sum = 0.f;
  for (int e = lane; e < E; e += 64) {
    const float p = expf(score[e] - top);
    score[e] = p;
    sum += p;
  }
  sum = wave_sum(sum);
  for (int e = lane; e < E; e += 64) {
    const float s = score[e] / sum;
    float c = s + (correction ? correction[e] : 0.f);
    c = c == c ? fmaxf(c, -3.0e38f) : -3.0e38f;   // (a taken expert is -inf)
    score[e] = s;
    choice[e] = c;
  }
  __syncthreads();
  if (E <= kRankedExperts) {   // (uniform)
    for (int e = lane; e < E; e += 64) {
      const float v = choice[e];
      int ahead = 0, o = 0;
      for (; o + 4 <= E; o += 4) {
        const f32x4 w = *reinterpret_cast<const f32x4*>(choice + o);
#pragma unroll
        for (int i = 0; i < 4; ++i) ahead += w[i] > v || (w[i] == v && o + i < e);
      }
      for (; o < E; ++o) ahead += choice[o] > v || (choice[o] == v && o < e);
      if (ahead < k) {
        sel[ahead] = score[e];
        topk_id[m * ld + ahead] = e;
      }
    }
    __syncthreads();
  }
  for (int j = 0; j < k && E > kRankedExperts; ++j) {
    float best = ninf;
    int bi = 0x7fffffff;
    for (int e = lane; e < E; e += 64)
      if (choice[e] > best) {
        best = choice[e];
        bi = e;
      }
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float ob = __shfl_xor(best, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (ob > best || (ob == best && oi < bi)) {
        best = ob;
        bi = oi;
      }
    }
    if (lane == 0) {
      sel[j] = score[bi];
      topk_id[m * ld + j] = bi;
      choice[bi] = ninf;
    }
    __syncthreads();
  }
  float total = 0.f;
  for (int j = lane; j < k; j += 64) total += sel[j];
  total = wave_sum(total) + 1e-20f;
  for (int j = lane; j < k; j += 64) topk_w[m * ld + j] = bad ? __builtin_nanf("") : sel[j] / total * scale;
}

}  // namespace

// tnx_residual_norm's descriptors with a centred norm, a factor, an extra row or the depth average (the caller has checked
// what they share with the others)
int tnx_internal_layer_step(hipStream_t st, const tnx_residual_norm_desc* d) {
  TNX_REQUIRE(d->mode <= 1 && d->groups <= 1 && !d->shift, "residual_norm: centred norms, a factor, extra rows and the depth average go with modes 0 and 1, one part and no shift");
  const bool extra = d->extra.ld > 0;
  TNX_REQUIRE(d->mode == 0 || (src_given(d->y) && d->y.ld >= d->D), "residual_norm: no incoming rows");
  TNX_REQUIRE(!extra || (d->mode == 1 && src_given(d->extra) && d->extra.ld >= d->D), "residual_norm: extra rows join incoming ones, and hold a row");
  TNX_REQUIRE(!d->hist || (d->hist_n >= 0 && d->hist_w && d->hist_plane >= d->M * d->D), "residual_norm: the depth average needs its weights and whole planes");
  TNX_REQUIRE(!d->hist || d->x_out || d->x != d->hist, "residual_norm: the average would overwrite an earlier result");
  TNX_REQUIRE(d->M < (int64_t)1 << 31, "residual_norm: too many rows");
  StepArgs a;
  memset(&a, 0, sizeof(a));
  a.D = d->D; a.eps = d->eps; a.w_offset = d->w_offset; a.mult = d->mult == 0.f ? 1.f : d->mult; a.mode = d->mode; a.w_post = d->w_post; a.x = d->x;
  a.x_out = d->x_out ? d->x_out : d->x;
  if (a.x_out == d->x && d->mode == 0 && !d->hist) a.x_out = nullptr;
  a.route_w = d->route_w; a.route_k = d->route_k; a.extra_w = d->extra_w; a.has_extra = extra;
  a.hist = d->hist; a.hist_plane = d->hist ? d->hist_plane : 0; a.hist_n = d->hist_n; a.hist_store = d->hist_store; a.hist_w = d->hist_w;
  a.w_next = d->w_next; a.out = d->out; a.out_ld = d->out_ld; a.out_frag = d->out_frag;
  auto run = [&](auto t) {
    using T = decltype(t);
    const RowSrc<T> y = row_src<T>(d->y), e = row_src<T>(d->extra);
    return d->center ? launch_step<true, T>(st, d->M, a, y, e) : launch_step<false, T>(st, d->M, a, y, e);
  };
  return d->dtype == TNX_BF16 ? run(uint16_t{}) : run(float{});
}

extern "C" int tnx_rownorm_kvwrite(void* stream, const tnx_rownorm_kvwrite_desc* d) {
  TNX_REQUIRE(d, "rownorm_kvwrite: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->T > 0 && d->S > 0 && d->H > 0 && d->G > 0 && d->H % d->G == 0 && d->B * d->T < (int64_t)1 << 31, "rownorm_kvwrite: bad shape");
  TNX_REQUIRE(d->dk > 0 && d->dv > 0 && d->dkp >= d->dk && d->dvp >= d->dv, "rownorm_kvwrite: bad head sizes");
  TNX_REQUIRE(src_given(d->y) && d->w_q && d->col_ptr && d->q_out && (!d->kcache == !d->vcache) && (!d->kcache || d->w_k), "rownorm_kvwrite: null pointer");
  TNX_REQUIRE(d->y.ld >= (int64_t)d->H * d->dk && (!d->kcache || (d->k_off >= 0 && d->v_off >= 0 && d->y.ld >= d->k_off + (int64_t)d->G * d->dk &&
                                                                  d->y.ld >= d->v_off + (int64_t)d->G * d->dv)),
              "rownorm_kvwrite: heads outside the row");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "rownorm_kvwrite: bad dtype %d", d->dtype);
  RowNormArgs a;
  a.T = d->T; a.S = d->S; a.H = d->H; a.G = d->G; a.dk = d->dk; a.dv = d->dv; a.dkp = d->dkp; a.dvp = d->dvp; a.eps = d->eps; a.w_q = d->w_q; a.w_k = d->w_k;
  a.k_off = d->k_off; a.v_off = d->v_off; a.col_ptr = d->col_ptr;
  if (d->dtype == TNX_BF16)
    return launch_rownorm_kv(as_stream(stream), d->B * d->T, a, row_src<uint16_t>(d->y), (uint16_t*)d->q_out, (uint16_t*)d->kcache, (uint16_t*)d->vcache);
  return launch_rownorm_kv(as_stream(stream), d->B * d->T, a, row_src<float>(d->y), (float*)d->q_out, (float*)d->kcache, (float*)d->vcache);
}

extern "C" int tnx_poly_norm(void* stream, int dtype, const tnx_rows_src* y, int64_t M, int64_t F, const float* coef, float eps, void* out,
                             int64_t out_ld, int out_frag) {
  TNX_REQUIRE(y && src_given(*y) && coef && out, "poly_norm: null pointer");
  TNX_REQUIRE(M > 0 && M < (int64_t)1 << 31 && F > 0 && y->ld >= F && out_ld >= F, "poly_norm: bad shape");
  TNX_REQUIRE(dtype == TNX_BF16 || dtype == TNX_F32, "poly_norm: bad dtype %d", dtype);
  if (dtype == TNX_BF16) return launch_poly(as_stream(stream), M, row_src<uint16_t>(*y), F, coef, eps, (uint16_t*)out, out_ld, out_frag);
  return launch_poly(as_stream(stream), M, row_src<float>(*y), F, coef, eps, (float*)out, out_ld, out_frag);
}

extern "C" int tnx_route_scores(void* stream, const tnx_rows_src* z, int64_t M, int E, int k, const float* correction, float scale, int64_t gate_off,
                                int ld, float* topk_w, int32_t* topk_id, float* gate_w) {
  TNX_REQUIRE(z && src_given(*z) && topk_w && topk_id, "route_scores: null pointer");
  TNX_REQUIRE(M > 0 && M < ((int64_t)1 << 31) && E > 0 && E <= 4096 && k > 0 && k <= E && z->ld >= E, "route_scores: bad shape E=%d k=%d", E, k);
  TNX_REQUIRE(ld >= k, "route_scores: %d entries per row for %d experts", ld, k);
  TNX_REQUIRE((!gate_w && ld == k) || (gate_off >= 0 && gate_off < z->ld), "route_scores: the gate lies outside the row");
  hipLaunchKernelGGL(route_scores_kernel, dim3((unsigned)M), dim3(64), (size_t)((E + 3) / 4 * 4 + E + k) * 4, as_stream(stream), row_src<float>(*z), E, k,
                     correction, scale, gate_off, ld, topk_w, topk_id, gate_w);
  TNX_CHECK_LAUNCH("route_scores");
  return TNX_OK;
}
