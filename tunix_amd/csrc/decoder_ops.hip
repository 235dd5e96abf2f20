// The small operations of decoders with dense weights and an fp32 residual stream: embedding,
// post-norm + residual + next pre-norm or token shift, parallel sublayers' residual + norm + input convolutions,
// partial rotation + cache write, convolution + cache write, gated norms, gated unit, the choice of experts, and the statistics / sampling of finished logits.  Norms, angles and the residual are 32-bit;
// matrix operands leave in the model's dtype (bf16 or fp32).
#include <string.h>

#include <mutex>
#include <type_traits>

#include "decoder.h"
#include "rng.h"

int tnx_internal_layer_step(hipStream_t st, const tnx_residual_norm_desc* d);

namespace {

__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  const int wave = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[wave] = v;
  __syncthreads();
  float s = 0.f;
  for (int w = 0; w < nw; ++w) s += red[w];
  return s;
}

// ---- embedding ---------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void embed_rows_kernel(const T* table, int64_t V, int64_t D, const int32_t* ids,
                                                         int64_t ids_ld, const int32_t* col_ptr, int64_t Tn, float scale, float* x,
                                                         T* cat, int64_t cat_ld, int64_t cat_off, int cat_frag, const T* pos,
                                                         int64_t n_pos, const int32_t* starts) {
  const int64_t row = blockIdx.x, b = row / Tn, t = row % Tn;
  const int col = col_ptr ? *col_ptr : 0;
  const int64_t p = pos ? min(max((int64_t)col + t - starts[b], (int64_t)0), n_pos - 1) : 0;
  int64_t id = ids[b * ids_ld + col + t];
  if (id < 0 || id >= V) id = 0;   // padding columns: never read by a later token
  if (D % 8 == 0 && cat_ld % 8 == 0) {   // (cat_off is then a multiple of eight, too, where cat is given)
    const RowSrc<T> src{table, nullptr, 1, 0, D};
    for (int64_t i = (int64_t)threadIdx.x * 8; i < D; i += 2048) {
      float f[8];
      get8(src, id, i, f);
      if (cat) put8(cat + (cat_frag ? frag_index(row, cat_off + i, cat_ld) : row * cat_ld + cat_off + i), f);
#pragma unroll
      for (int j = 0; j < 8; ++j) f[j] *= scale;
      if (pos) {
        float g[8];
        get8(RowSrc<T>{pos, nullptr, 1, 0, D}, p, i, g);
#pragma unroll
        for (int j = 0; j < 8; ++j) f[j] += g[j];
      }
      put8(x + row * D + i, f);
    }
    return;
  }
  for (int64_t i = threadIdx.x; i < D; i += 256) {
    const T v = table[id * D + i];
    x[row * D + i] = scale * ld_elem(&v, 0) + (pos ? ld_elem(pos, p * D + i) : 0.f);
    if (cat) cat[cat_frag ? frag_index(row, cat_off + i, cat_ld) : row * cat_ld + cat_off + i] = v;
  }
}

// ---- residual + norms --------------------------------------------------------------------------
struct ResNormArgs {
  int64_t M, D;
  float eps, w_offset;
  const void* y;
  const float* ws;
  int split;
  int64_t plane, y_ld;
  int mode;               // 0: nothing arrives, 1: x += norm(y) . w_post, 2: x = y, 3: x = norm(x) . w_post
  const float* w_post;
  float* x;
  // rows_kernel: norms in equal parts of a row, routed rows, token shift
  int groups;
  float* x_out;
  const float* route_w;   // [M, route_k]: y holds route_k rows per row of x, summed with these weights
  int route_k;
  const float* shift;     // [D]: out = x + (x of the token before - x) . shift
  float* before;          // [B, D]: x of the last token of the call before
  const int32_t* starts;
  const int32_t* col_ptr;
  int64_t B, T;
  int run;                // tokens of a work-group
  const float* w_next;    // null: out = x in the model's dtype
  void* out;
  int64_t out_ld;
  int out_frag;
};

// any D that fits LDS
template <typename T>
__global__ __launch_bounds__(256) void resnorm_kernel(const ResNormArgs a) {
  extern __shared__ __align__(16) float hrow[];
  __shared__ float red[4];
  const int64_t row = blockIdx.x;
  const RowSrc<T> src{reinterpret_cast<const T*>(a.y), a.ws, a.ws ? max(a.split, 2) : 1, a.plane, a.y_ld};
  auto incoming = [&](int64_t i) {
    if (!a.ws) return src.get(row, i);
    float v = 0.f;
    for (int z = 0; z < a.split; ++z) v += a.ws[z * a.plane + row * a.y_ld + i];
    return v;
  };
  float ss = 0.f;
  if (a.mode != 0)
    for (int64_t i = threadIdx.x; i < a.D; i += 256) {
      const float v = incoming(i);
      hrow[i] = v;
      ss += v * v;
    }
  float r = 1.f;
  if (a.mode == 1) r = 1.0f / sqrtf(block_sum(ss, red) / (float)a.D + a.eps);
  ss = 0.f;
  for (int64_t i = threadIdx.x; i < a.D; i += 256) {
    float h;
    if (a.mode == 1) h = a.x[row * a.D + i] + hrow[i] * r * (a.w_offset + a.w_post[i]);
    else if (a.mode == 2) h = hrow[i];
    else h = a.x[row * a.D + i];
    if (a.mode != 0) a.x[row * a.D + i] = h;
    hrow[i] = h;
    ss += h * h;
  }
  float rn = 1.f;
  if (a.w_next) rn = 1.0f / sqrtf(block_sum(ss, red) / (float)a.D + a.eps);
  T* out = reinterpret_cast<T*>(a.out);
  for (int64_t i = threadIdx.x; i < a.D; i += 256) {
    const float v = a.w_next ? hrow[i] * rn * (a.w_offset + a.w_next[i]) : hrow[i];
    st_elem(out, a.out_frag ? frag_index(row, i, a.out_ld) : row * a.out_ld + i, v);
  }
}

// D % 8 == 0: eight elements per thread and turn, the row stays in registers.  Everything the row needs
// -- residual, incoming values, both weights -- is requested before the first sum: the kernel is one
// memory round trip and two block reductions long.
template <int MAXC, typename T>
__global__ __launch_bounds__(256) void resnorm_vec_kernel(const ResNormArgs a) {
  __shared__ float red[4];
  const int64_t row = blockIdx.x;
  const int nch = (int)(a.D / 8);
  // (mode and w_next are the same for the whole grid: uniform branches)
  const RowSrc<T> src{reinterpret_cast<const T*>(a.y), a.ws, a.split, a.plane, a.y_ld};
  float h[MAXC][8], xo[MAXC][8], wp[MAXC][8], wn[MAXC][8];
  auto load8f = [](const float* p, float (&f)[8]) {
    const f32x4 u = *reinterpret_cast<const f32x4*>(p), v = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      f[j] = u[j];
      f[4 + j] = v[j];
    }
  };
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int64_t col = (int64_t)min(c * 256 + (int)threadIdx.x, nch - 1) * 8;
    if (a.mode != 2) load8f(a.x + row * a.D + col, xo[c]);
    if (a.mode == 1) load8f(a.w_post + col, wp[c]);
    if (a.w_next) load8f(a.w_next + col, wn[c]);
    if (a.mode != 0) {
      if (a.ws && a.split == 1) load8f(a.ws + row * a.y_ld + col, h[c]);
      else get8(src, row, col, h[c]);
    }
  }
  float ss = 0.f;
  float r = 1.f;
  if (a.mode == 1) {
#pragma unroll
    for (int c = 0; c < MAXC; ++c)
      if (c * 256 + (int)threadIdx.x < nch)
#pragma unroll
        for (int j = 0; j < 8; ++j) ss += h[c][j] * h[c][j];
    r = 1.0f / sqrtf(block_sum(ss, red) / (float)a.D + a.eps);
  }
  ss = 0.f;
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int ch = c * 256 + threadIdx.x;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      if (a.mode == 1) h[c][j] = xo[c][j] + h[c][j] * r * (a.w_offset + wp[c][j]);
      else if (a.mode == 0) h[c][j] = xo[c][j];
    }
    if (ch < nch) {
#pragma unroll
      for (int j = 0; j < 8; ++j) ss += h[c][j] * h[c][j];
      if (a.mode != 0) put8(a.x + row * a.D + (int64_t)ch * 8, h[c]);
    }
  }
  float rn = 1.f;
  if (a.w_next) rn = 1.0f / sqrtf(block_sum(ss, red) / (float)a.D + a.eps);
  T* out = reinterpret_cast<T*>(a.out);
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int ch = c * 256 + threadIdx.x;
    if (ch >= nch) continue;
    const int64_t col = (int64_t)ch * 8;
    if (a.w_next)
#pragma unroll
      for (int j = 0; j < 8; ++j) h[c][j] = h[c][j] * rn * (a.w_offset + wn[c][j]);
    put8(out + (a.out_frag ? frag_index(row, col, a.out_ld) : row * a.out_ld + col), h[c]);
  }
}

// 1 / sqrt(mean + eps) of equal parts of a row whose elements the threads own in runs: part[i] is the
// sum of squares of run i, `per` runs (of `len / per` elements) make a part.  Two barriers; the result is in gs[part].
__device__ __forceinline__ void part_scales(const float* part, float* gs, int groups, int per, float len, float eps) {
  __syncthreads();
  const int lane = threadIdx.x & 63, nw = blockDim.x >> 6;
  for (int g = threadIdx.x >> 6; g < groups; g += nw) {
    float s = 0.f;
    for (int i = lane; i < per; i += 64) s += part[g * per + i];
    s = wave_sum(s);
    if (lane == 0) gs[g] = 1.0f / sqrtf(s / len + eps);
  }
  __syncthreads();
}

// The general residual step: norms over equal parts of a row, weighted sums of routed rows, token shift.
// A work-group walks `run` tokens of one sequence; with a shift it forms the token before its first one
// as well (x and x_out are then different buffers, unless the call brings one token per sequence).
template <int NT, int MAXC, bool ROUTES, typename T>   // NT threads, MAXC runs of eight per thread
__global__ __launch_bounds__(NT) void resnorm_rows_kernel(const ResNormArgs a) {
  __shared__ float red[NT / 64], part[MAXC * NT], gs[MAXC * NT];
  const int64_t runs = (a.T + a.run - 1) / a.run, b = blockIdx.x / runs, t0 = blockIdx.x % runs * a.run;
  const int64_t t1 = min(a.T, t0 + a.run);
  const int nch = (int)(a.D / 8), per = nch / a.groups, tid = threadIdx.x;
  const int col0 = a.shift ? *a.col_ptr : 0, start = a.shift ? a.starts[b] : 0;
  const RowSrc<T> src{reinterpret_cast<const T*>(a.y), a.ws, a.split, a.plane, a.y_ld};
  float wp[MAXC][8], wn[MAXC][8], prev[MAXC][8], h[MAXC][8];
  auto load8f = [](const float* p, float (&f)[8]) {
    const f32x4 u = *reinterpret_cast<const f32x4*>(p), v = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      f[j] = u[j];
      f[4 + j] = v[j];
    }
  };
  const float* wnext = a.shift ? a.shift : a.w_next;
  auto column = [&](int c) { return (int64_t)min(c * NT + tid, nch - 1) * 8; };
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    if (a.w_post) load8f(a.w_post + column(c), wp[c]);
    if (wnext) load8f(wnext + column(c), wn[c]);
#pragma unroll
    for (int j = 0; j < 8; ++j) prev[c][j] = 0.f;
    if (a.shift && t0 == 0 && col0 > start) load8f(a.before + b * a.D + column(c), prev[c]);
  }
  float r[MAXC];
  auto scales = [&](const float (&v)[MAXC][8]) {
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      if (c * NT + tid >= nch) continue;
      float q = 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) q += v[c][j] * v[c][j];
      ss += q;
      if (a.groups > 1) part[c * NT + tid] = q;
    }
    if (a.groups == 1) {
      const float s = 1.0f / sqrtf(block_sum(ss, red) / (float)a.D + a.eps);
#pragma unroll
      for (int c = 0; c < MAXC; ++c) r[c] = s;
      return;
    }
    part_scales(part, gs, a.groups, per, (float)(per * 8), a.eps);
#pragma unroll
    for (int c = 0; c < MAXC; ++c) r[c] = gs[min(c * NT + tid, nch - 1) / per];
  };
  for (int64_t t = a.shift && t0 > 0 ? t0 - 1 : t0; t < t1; ++t) {
    const int64_t row = b * a.T + t;
    float xo[MAXC][8];
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      const int64_t col = column(c);
      if (a.mode != 2) load8f(a.x + row * a.D + col, xo[c]);
      if (a.mode == 1 || a.mode == 2) {
        if constexpr (ROUTES) {
#pragma unroll
          for (int j = 0; j < 8; ++j) h[c][j] = 0.f;
#pragma unroll 4
          for (int k = 0; k < a.route_k; ++k) {
            const float w = a.route_w[row * a.route_k + k];
            float f[8];
            get8(RowSrc<T>{src.y, nullptr, 1, 0, a.y_ld}, row * a.route_k + k, col, f);
#pragma unroll
            for (int j = 0; j < 8; ++j) h[c][j] += w * f[j];
          }
        } else if (a.ws && a.split == 1) {
          load8f(a.ws + row * a.y_ld + col, h[c]);
        } else {
          get8(src, row, col, h[c]);
        }
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) h[c][j] = xo[c][j];
      }
    }
    if (a.mode == 1 || a.mode == 3) {
      scales(h);
#pragma unroll
      for (int c = 0; c < MAXC; ++c)
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float v = h[c][j] * r[c] * (a.w_offset + wp[c][j]);
          h[c][j] = a.mode == 1 ? xo[c][j] + v : v;
        }
    }
    if (t >= t0) {
      if (a.w_next) scales(h);   // (uniform)
      T* out = reinterpret_cast<T*>(a.out);
#pragma unroll
      for (int c = 0; c < MAXC; ++c) {
        if (c * NT + tid >= nch) continue;
        const int64_t col = column(c);
        if (a.mode != 0 || a.x_out != a.x) put8(a.x_out + row * a.D + col, h[c]);
        float o[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          o[j] = h[c][j];
          if (a.shift) o[j] = h[c][j] + ((col0 + t > start ? prev[c][j] : 0.f) - h[c][j]) * wn[c][j];
          else if (a.w_next) o[j] = h[c][j] * r[c] * (a.w_offset + wn[c][j]);
        }
        put8(out + (a.out_frag ? frag_index(row, col, a.out_ld) : row * a.out_ld + col), o);
      }
    }
#pragma unroll
    for (int c = 0; c < MAXC; ++c)
#pragma unroll
      for (int j = 0; j < 8; ++j) prev[c][j] = h[c][j];
  }
  if (a.shift && a.T == 1)
#pragma unroll
    for (int c = 0; c < MAXC; ++c)
      if (c * NT + tid < nch) put8(a.before + b * a.D + column(c), h[c]);
}

// the same for any D that fits LDS twice: h and the token before, a thread owning the columns tid + 256 i
template <typename T>
__global__ __launch_bounds__(256) void resnorm_rows_any_kernel(const ResNormArgs a) {
  extern __shared__ __align__(16) float hrow[];
  float* prev = hrow + a.D;
  __shared__ float gs[1024];
  const int64_t runs = (a.T + a.run - 1) / a.run, b = blockIdx.x / runs, t0 = blockIdx.x % runs * a.run;
  const int64_t t1 = min(a.T, t0 + a.run);
  const int per = (int)(a.D / a.groups), tid = threadIdx.x, lane = tid & 63;
  const int col0 = a.shift ? *a.col_ptr : 0, start = a.shift ? a.starts[b] : 0;
  const RowSrc<T> src{reinterpret_cast<const T*>(a.y), a.ws, a.split, a.plane, a.y_ld};
  auto scales = [&]() {
    __syncthreads();
    for (int g = tid >> 6; g < a.groups; g += 4) {
      float s = 0.f;
      for (int i = lane; i < per; i += 64) s += hrow[g * per + i] * hrow[g * per + i];
      s = wave_sum(s);
      if (lane == 0) gs[g] = 1.0f / sqrtf(s / (float)per + a.eps);
    }
    __syncthreads();
  };
  for (int64_t i = tid; i < a.D; i += 256) prev[i] = a.shift && t0 == 0 && col0 > start ? a.before[b * a.D + i] : 0.f;
  for (int64_t t = a.shift && t0 > 0 ? t0 - 1 : t0; t < t1; ++t) {
    const int64_t row = b * a.T + t;
    for (int64_t i = tid; i < a.D; i += 256) {
      float v = 0.f;
      if (a.mode == 0 || a.mode == 3) v = a.x[row * a.D + i];
      else if (a.route_w)
        for (int k = 0; k < a.route_k; ++k) v += a.route_w[row * a.route_k + k] * src.get(row * a.route_k + k, i);
      else if (a.ws && a.split == 1) v = a.ws[row * a.y_ld + i];
      else v = src.get(row, i);
      hrow[i] = v;
    }
    if (a.mode == 1 || a.mode == 3) {
      scales();
      for (int64_t i = tid; i < a.D; i += 256) {
        const float v = hrow[i] * gs[i / per] * (a.w_offset + a.w_post[i]);
        hrow[i] = a.mode == 1 ? a.x[row * a.D + i] + v : v;
      }
    }
    if (t >= t0) {
      if (a.w_next) scales();
      T* out = reinterpret_cast<T*>(a.out);
      for (int64_t i = tid; i < a.D; i += 256) {
        const float h = hrow[i];
        if (a.mode != 0 || a.x_out != a.x) a.x_out[row * a.D + i] = h;
        float o = h;
        if (a.shift) o = h + ((col0 + t > start ? prev[i] : 0.f) - h) * a.shift[i];
        else if (a.w_next) o = h * gs[i / per] * (a.w_offset + a.w_next[i]);
        st_elem(out, a.out_frag ? frag_index(row, i, a.out_ld) : row * a.out_ld + i, o);
      }
    }
    __syncthreads();   // every group's sums have read hrow
    for (int64_t i = tid; i < a.D; i += 256) prev[i] = hrow[i];
  }
  if (a.shift && a.T == 1)
    for (int64_t i = tid; i < a.D; i += 256) a.before[b * a.D + i] = prev[i];
}

template <typename T>
int launch_resnorm_rows(hipStream_t st, ResNormArgs a) {
  a.run = 8;
  while (a.run > 1 && a.B * cdiv(a.T, a.run) < 1024) a.run /= 2;
  const dim3 grid((unsigned)(a.B * cdiv(a.T, a.run)));
  const bool vec = a.D % 8 == 0 && a.D / a.groups % 8 == 0 && a.y_ld % 8 == 0 && a.out_ld % 8 == 0 && a.plane % 8 == 0;
  if (!vec) {
    TNX_REQUIRE(a.D <= 7168 && a.groups <= 1024, "residual_norm: D=%lld in %d parts needs runs of eight", (long long)a.D, a.groups);
    hipLaunchKernelGGL((resnorm_rows_any_kernel<T>), grid, dim3(256), (size_t)a.D * 8, st, a);
    return TNX_OK;
  }
  auto launch = [&](auto routes) {
    constexpr bool R = decltype(routes)::value;
    if (a.D <= 2048) hipLaunchKernelGGL((resnorm_rows_kernel<256, 1, R, T>), grid, dim3(256), 0, st, a);
    else if (a.D <= 4096) hipLaunchKernelGGL((resnorm_rows_kernel<512, 1, R, T>), grid, dim3(512), 0, st, a);
    else if (a.D <= 8192) hipLaunchKernelGGL((resnorm_rows_kernel<1024, 1, R, T>), grid, dim3(1024), 0, st, a);
    else hipLaunchKernelGGL((resnorm_rows_kernel<1024, 2, R, T>), grid, dim3(1024), 0, st, a);
  };
  if (a.route_w) launch(std::true_type{});
  else launch(std::false_type{});
  return TNX_OK;
}

template <typename T>
void launch_resnorm(hipStream_t st, const ResNormArgs& a) {
  const bool vec = a.D % 8 == 0 && a.y_ld % 8 == 0 && a.out_ld % 8 == 0 && a.plane % 8 == 0;
  const dim3 grid((unsigned)a.M);
  if (!vec) hipLaunchKernelGGL((resnorm_kernel<T>), grid, dim3(256), (size_t)a.D * 4, st, a);
  else if (a.D <= 2048) hipLaunchKernelGGL((resnorm_vec_kernel<1, T>), grid, dim3(256), 0, st, a);
  else if (a.D <= 4096) hipLaunchKernelGGL((resnorm_vec_kernel<2, T>), grid, dim3(256), 0, st, a);
  else if (a.D <= 8192) hipLaunchKernelGGL((resnorm_vec_kernel<4, T>), grid, dim3(256), 0, st, a);
  else hipLaunchKernelGGL((resnorm_vec_kernel<8, T>), grid, dim3(256), 0, st, a);
}

// ---- layers whose sublayers read one norm: residual + norm + input convolutions --------------------
struct ParallelArgs {
  int64_t D, B, T;
  float eps, mult;
  int n_in;
  const void* y[3];
  const float* ws[3];
  int split[3];
  int64_t plane[3], y_ld[3];
  const float* w_post[3];
  float y_scale[3];
  const float* x;
  float* x_out;
  const float* add;
  const float* w_next;
  int taps, slots;
  const float* conv1;
  const float* conv2;
  void* out1;
  void* out2;
  int64_t out_ld;
  int out_frag;
  float* ring;
  float* tail;
  const int32_t* starts;
  const int32_t* col_ptr;
  int run;                // tokens of a work-group
};
// eight values of a row as they lie in memory
template <typename T>
struct Raw8;
template <>
struct Raw8<uint16_t> {
  u32x4 v;
  __device__ __forceinline__ void load(const uint16_t* p) { v = *reinterpret_cast<const u32x4*>(p); }
  __device__ __forceinline__ void get(float (&f)[8]) const {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      f[2 * j] = bflo(v[j]);
      f[2 * j + 1] = bfhi(v[j]);
    }
  }
};
template <>
struct Raw8<float> {
  f32x4 v[2];
  __device__ __forceinline__ void load(const float* p) {
    v[0] = *reinterpret_cast<const f32x4*>(p);
    v[1] = *reinterpret_cast<const f32x4*>(p + 4);
  }
  __device__ __forceinline__ void get(float (&f)[8]) const {
#pragma unroll
    for (int j = 0; j < 8; ++j) f[j] = v[j >> 2][j & 3];
  }
};

// A work-group walks `run` tokens of one sequence; it forms h of the taps - 1 tokens in front of them as well, or
// takes it from the ring where they belong to an earlier call.  A thread owns runs of eight columns.  The next
// token's rows are requested before this one's sums (PLANES: incoming rows in partial planes, one token at a time).
template <int NT, int MAXC, int TAPS, bool PLANES, typename T>
__global__ __launch_bounds__(NT) void parallel_step_kernel(const ParallelArgs a) {
  constexpr int NW = NT / 64;
  __shared__ float red[2][NW][3];   // (two reductions a token take turns: one barrier each)
  const int64_t runs = (a.T + a.run - 1) / a.run, b = blockIdx.x / runs, t0 = blockIdx.x % runs * a.run;
  const int64_t t1 = min(a.T, t0 + a.run);
  const int nch = (int)(a.D / 8), tid = threadIdx.x, wave = tid >> 6;
  const bool conv = a.conv1 != nullptr;
  const int col0 = conv ? *a.col_ptr : 0, start = conv ? a.starts[b] : 0;
  auto column = [&](int c) { return (int64_t)min(c * NT + tid, nch - 1) * 8; };
  auto load8f = [](const float* p, float (&f)[8]) {
    Raw8<float> r;
    r.load(p);
    r.get(f);
  };
  struct Rows {
    Raw8<float> x[MAXC];
    Raw8<T> y[3][MAXC];
  };
  auto request = [&](int64_t row, Rows& r) {
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      r.x[c].load(a.x + row * a.D + column(c));
      if constexpr (!PLANES)
#pragma unroll
        for (int p = 0; p < 3; ++p)
          if (p < a.n_in) r.y[p][c].load(reinterpret_cast<const T*>(a.y[p]) + row * a.y_ld[p] + column(c));
    }
  };
  const int64_t first = conv ? t0 - (TAPS - 1) : t0, tb = max(first, (int64_t)0);
  Rows cur, nxt;
  request(b * a.T + tb, cur);
  float wn[MAXC][8], wp[2][MAXC][8], c1[TAPS][MAXC][8], c2[TAPS][MAXC][8], prev[TAPS][MAXC][8];   // prev[j]: h of j + 1 tokens before
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    load8f(a.w_next + column(c), wn[c]);
#pragma unroll
    for (int p = 0; p < 2; ++p)
      if (a.w_post[p]) load8f(a.w_post[p] + column(c), wp[p][c]);
#pragma unroll
    for (int k = 0; k < TAPS; ++k) {
      if (conv) load8f(a.conv1 + k * a.D + column(c), c1[k][c]);
      if (a.conv2) load8f(a.conv2 + k * a.D + column(c), c2[k][c]);
#pragma unroll
      for (int j = 0; j < 8; ++j) prev[k][c][j] = 0.f;
    }
  }
#pragma unroll
  for (int k = 0; k + 1 < TAPS; ++k) {   // tokens of an earlier call
    const int64_t t = tb - 1 - k;
    if (conv && t < 0 && col0 + t >= start)
#pragma unroll
      for (int c = 0; c < MAXC; ++c) load8f(a.ring + (b * a.slots + (col0 + t) % a.slots) * a.D + column(c), prev[k][c]);
  }
  for (int64_t t = tb; t < t1; ++t) {
    const int64_t row = b * a.T + t;
    const bool live = col0 + t >= start;   // (uniform) otherwise h counts as zero for the tokens behind
    float h[MAXC][8], in[3][MAXC][8], s[3] = {0.f, 0.f, 0.f};
    if constexpr (!PLANES) request(b * a.T + min(t + 1, t1 - 1), nxt);
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      cur.x[c].get(h[c]);
#pragma unroll
      for (int p = 0; p < 3; ++p) {
        if (p >= a.n_in) continue;
        if constexpr (PLANES) get8(RowSrc<T>{reinterpret_cast<const T*>(a.y[p]), a.ws[p], a.split[p], a.plane[p], a.y_ld[p]}, row, column(c), in[p][c]);
        else cur.y[p][c].get(in[p][c]);
        if (a.w_post[p] && c * NT + tid < nch)
#pragma unroll
          for (int j = 0; j < 8; ++j) s[p] += in[p][c][j] * in[p][c][j];
      }
    }
    if (a.n_in > 0) {   // (uniform)
#pragma unroll
      for (int p = 0; p < 3; ++p)
        if (p < a.n_in && a.w_post[p]) {
          s[p] = wave_sum(s[p]);
          if ((tid & 63) == 0) red[0][wave][p] = s[p];
        }
      __syncthreads();
#pragma unroll
      for (int p = 0; p < 3; ++p) {
        if (p >= a.n_in) continue;
        float f = a.mult * a.y_scale[p];
        if (a.w_post[p]) {
          float sum = 0.f;
#pragma unroll
          for (int w = 0; w < NW; ++w) sum += red[0][w][p];
          f *= 1.0f / sqrtf(sum / (float)a.D + a.eps);
        }
#pragma unroll
        for (int c = 0; c < MAXC; ++c) {
          float w2[8];
          if (p == 2 && a.w_post[2]) load8f(a.w_post[2] + column(c), w2);
#pragma unroll
          for (int j = 0; j < 8; ++j) h[c][j] += f * in[p][c][j] * (a.w_post[p] ? (p == 2 ? w2[j] : wp[p & 1][c][j]) : 1.f);
        }
      }
    }
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      if (a.add) {
        float v[8];
        load8f(a.add + column(c), v);
#pragma unroll
        for (int j = 0; j < 8; ++j) h[c][j] += v[j];
      }
      if (c * NT + tid < nch) {
        if (a.x_out && t >= t0) put8(a.x_out + row * a.D + column(c), h[c]);
#pragma unroll
        for (int j = 0; j < 8; ++j) ss += h[c][j] * h[c][j];
      }
    }
    ss = wave_sum(ss);
    if ((tid & 63) == 0) red[1][wave][0] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) ss += red[1][w][0];
    const float rn = 1.0f / sqrtf(ss / (float)a.D + a.eps);
#pragma unroll
    for (int c = 0; c < MAXC; ++c)
#pragma unroll
      for (int j = 0; j < 8; ++j) h[c][j] *= rn * wn[c][j];
    if (t >= t0) {
#pragma unroll
      for (int c = 0; c < MAXC; ++c) {
        if (c * NT + tid >= nch) continue;
        const int64_t col = column(c), at = a.out_frag ? frag_index(row, col, a.out_ld) : row * a.out_ld + col;
        float o[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) o[j] = h[c][j];
        if (conv) {
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            o[j] += c1[TAPS - 1][c][j] * h[c][j];
#pragma unroll
            for (int k = 0; k + 1 < TAPS; ++k) o[j] += c1[TAPS - 2 - k][c][j] * prev[k][c][j];
          }
        }
        put8(reinterpret_cast<T*>(a.out1) + at, o);
        if (a.out2) {
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            o[j] = h[c][j] + c2[TAPS - 1][c][j] * h[c][j];
#pragma unroll
            for (int k = 0; k + 1 < TAPS; ++k) o[j] += c2[TAPS - 2 - k][c][j] * prev[k][c][j];
          }
          put8(reinterpret_cast<T*>(a.out2) + at, o);
        }
        if (TAPS > 1 && conv) {
          const int64_t keep = min(a.T, (int64_t)TAPS - 1);
          if (a.T == 1) put8(a.ring + (b * a.slots + col0 % a.slots) * a.D + col, h[c]);
          else if (t >= a.T - keep) put8(a.tail + (b * keep + t - (a.T - keep)) * a.D + col, h[c]);
        }
      }
    }
#pragma unroll
    for (int c = 0; c < MAXC; ++c)
#pragma unroll
      for (int j = 0; j < 8; ++j) {
#pragma unroll
        for (int k = TAPS - 1; k > 0; --k) prev[k][c][j] = prev[k - 1][c][j];
        prev[0][c][j] = live ? h[c][j] : 0.f;
      }
    if constexpr (PLANES) {
      if (t + 1 < t1) request(b * a.T + t + 1, cur);
    } else {
      cur = nxt;
    }
  }
}

__device__ __forceinline__ void block_sum2(float& a, float& b, float (*red)[2]) {
  a = wave_sum(a);
  b = wave_sum(b);
  const int wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
  __syncthreads();
  if ((threadIdx.x & 63) == 0) {
    red[wave][0] = a;
    red[wave][1] = b;
  }
  __syncthreads();
  a = b = 0.f;
  for (int w = 0; w < nw; ++w) {
    a += red[w][0];
    b += red[w][1];
  }
}

// the same for any width and number of taps that fit LDS: a ring of `taps` rows of h, a thread owning the columns
// tid + 256 i
template <typename T>
__global__ __launch_bounds__(256) void parallel_step_any_kernel(const ParallelArgs a) {
  extern __shared__ __align__(16) float hbuf[];
  __shared__ float red[4][2];
  const int64_t runs = (a.T + a.run - 1) / a.run, b = blockIdx.x / runs, t0 = blockIdx.x % runs * a.run;
  const int64_t t1 = min(a.T, t0 + a.run);
  const int tid = threadIdx.x, taps = a.conv1 ? a.taps : 1;
  const int col0 = a.conv1 ? *a.col_ptr : 0, start = a.conv1 ? a.starts[b] : 0;
  const int64_t first = t0 - (taps - 1);
  for (int64_t t = first; t < t1; ++t) {
    const bool live = col0 + t >= start;
    float* hr = hbuf + (t - first) % taps * a.D;
    if (t < 0) {
      for (int64_t i = tid; i < a.D; i += 256) hr[i] = live ? a.ring[(b * a.slots + (col0 + t) % a.slots) * a.D + i] : 0.f;
      continue;
    }
    const int64_t row = b * a.T + t;
    auto incoming = [&](int p, int64_t i) {
      return RowSrc<T>{reinterpret_cast<const T*>(a.y[p]), a.ws[p], a.split[p], a.plane[p], a.y_ld[p]}.get(row, i);
    };
    float r[3] = {1.f, 1.f, 1.f};
    for (int p = 0; p < a.n_in; ++p) {
      if (!a.w_post[p]) continue;
      float s = 0.f, z = 0.f;
      for (int64_t i = tid; i < a.D; i += 256) {
        const float v = incoming(p, i);
        s += v * v;
      }
      block_sum2(s, z, red);
      r[p] = 1.0f / sqrtf(s / (float)a.D + a.eps);
    }
    float ss = 0.f, z = 0.f;
    for (int64_t i = tid; i < a.D; i += 256) {
      float v = a.x[row * a.D + i];
      for (int p = 0; p < a.n_in; ++p) v += a.mult * a.y_scale[p] * (incoming(p, i) * (a.w_post[p] ? r[p] * a.w_post[p][i] : 1.f));
      if (a.add) v += a.add[i];
      if (a.x_out && t >= t0) a.x_out[row * a.D + i] = v;
      hr[i] = v;
      ss += v * v;
    }
    block_sum2(ss, z, red);
    const float rn = 1.0f / sqrtf(ss / (float)a.D + a.eps);
    for (int64_t i = tid; i < a.D; i += 256) {
      const float h = hr[i] * (rn * a.w_next[i]);
      hr[i] = live ? h : 0.f;
      if (t < t0) continue;
      const int64_t at = a.out_frag ? frag_index(row, i, a.out_ld) : row * a.out_ld + i;
      float o1 = h, o2 = h;
      if (a.conv1)
        for (int k = 0; k < taps; ++k) {
          const float u = k == 0 ? h : hbuf[(t - k - first) % taps * a.D + i];
          o1 += a.conv1[(int64_t)(taps - 1 - k) * a.D + i] * u;
          if (a.conv2) o2 += a.conv2[(int64_t)(taps - 1 - k) * a.D + i] * u;
        }
      st_elem(reinterpret_cast<T*>(a.out1), at, o1);
      if (a.out2) st_elem(reinterpret_cast<T*>(a.out2), at, o2);
      if (taps > 1) {
        const int64_t keep = min(a.T, (int64_t)taps - 1);
        if (a.T == 1) a.ring[(b * a.slots + col0 % a.slots) * a.D + i] = h;
        else if (t >= a.T - keep) a.tail[(b * keep + t - (a.T - keep)) * a.D + i] = h;
      }
    }
  }
}

template <int NT, int MAXC, bool PLANES, typename T>
void launch_parallel_taps(hipStream_t st, const ParallelArgs& a, const dim3& grid) {
  const int taps = a.conv1 ? a.taps : 1;
  if (taps == 1) hipLaunchKernelGGL((parallel_step_kernel<NT, MAXC, 1, PLANES, T>), grid, dim3(NT), 0, st, a);
  else if (taps == 2) hipLaunchKernelGGL((parallel_step_kernel<NT, MAXC, 2, PLANES, T>), grid, dim3(NT), 0, st, a);
  else if (taps == 3) hipLaunchKernelGGL((parallel_step_kernel<NT, MAXC, 3, PLANES, T>), grid, dim3(NT), 0, st, a);
  else hipLaunchKernelGGL((parallel_step_kernel<NT, MAXC, 4, PLANES, T>), grid, dim3(NT), 0, st, a);
}
template <int NT, int MAXC, typename T>
void launch_parallel_planes(hipStream_t st, const ParallelArgs& a, const dim3& grid) {
  bool planes = false;
  for (int p = 0; p < a.n_in; ++p) planes = planes || a.split[p] > 1;
  if (planes) launch_parallel_taps<NT, MAXC, true, T>(st, a, grid);
  else launch_parallel_taps<NT, MAXC, false, T>(st, a, grid);
}
constexpr size_t kParallelLds = 144 * 1024;
template <typename T>
int launch_parallel(hipStream_t st, ParallelArgs a) {
  a.run = 16;
  while (a.run > 1 && a.B * cdiv(a.T, a.run) < 1024) a.run /= 2;
  const dim3 grid((unsigned)(a.B * cdiv(a.T, a.run)));
  bool vec = a.D % 8 == 0 && a.D <= 8192 && a.out_ld % 8 == 0 && (!a.conv1 || a.taps <= 4);
  for (int p = 0; p < a.n_in; ++p) vec = vec && a.y_ld[p] % 8 == 0 && a.plane[p] % 8 == 0;
  if (!vec) {
    const size_t lds = (size_t)a.D * (a.conv1 ? a.taps : 1) * 4;
    TNX_REQUIRE(lds <= kParallelLds, "parallel_step: D=%lld with %d taps does not fit LDS", (long long)a.D, a.taps);
    static std::once_flag once;
    static hipError_t e = hipSuccess;
    std::call_once(once, [] {
      e = hipFuncSetAttribute(reinterpret_cast<const void*>(&parallel_step_any_kernel<T>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)kParallelLds);
    });
    if (e != hipSuccess) {
      tnx_set_error("parallel_step: cannot raise the dynamic LDS limit: %s", hipGetErrorString(e));
      return TNX_ELAUNCH;
    }
    hipLaunchKernelGGL((parallel_step_any_kernel<T>), grid, dim3(256), lds, st, a);
  } else if (a.D <= 2048) launch_parallel_planes<256, 1, T>(st, a, grid);
  else if (a.D <= 4096) launch_parallel_planes<512, 1, T>(st, a, grid);
  else launch_parallel_planes<512, 2, T>(st, a, grid);
  TNX_CHECK_LAUNCH("parallel_step");
  return TNX_OK;
}

// ---- short convolution of q, k and v, query temperature, value norm, cache write ----------------------
struct ConvKvArgs {
  int64_t B, T, S;
  int H, G, dk, dv, dkp, dvp, taps, slots;
  float coef, every, eps;
  int value_norm;
  int64_t off, C, q_off, k_off, v_off;
  const float* w;          // [taps, C]
  void* ring;              // [B, slots, C]
  const int32_t* starts;
  const int32_t* col_ptr;
  int run, lanes;          // vec: tokens of a lane group, lanes of a head
};
__device__ __forceinline__ float query_temperature(int pos, float coef, float every) {
  return 1.0f + coef * logf(floorf((float)(pos + 1) / every) + 1.0f);
}

template <typename T>
__global__ __launch_bounds__(256) void conv_kvwrite_kernel(const ConvKvArgs a, const RowSrc<T> src, T* q_out, T* kc, T* vc) {
  extern __shared__ __align__(16) float vals[];   // v [G, dv], then its heads' scales [G]
  float* vs = vals + a.G * a.dv;
  const int64_t row = blockIdx.x, b = row / a.T, t = row % a.T;
  const int tid = threadIdx.x, col0 = *a.col_ptr, start = a.starts[b], slot = col0 + (int)t;
  if (slot >= a.S) return;                                    // (uniform; the host sizes the cache)
  T* ring = reinterpret_cast<T*>(a.ring) + b * a.slots * a.C;
  auto convolved = [&](int64_t c) {
    float v = 0.f;
    for (int j = a.taps - 1; j >= 0; --j) {
      const int64_t col = (int64_t)slot - j;
      if (col < start) continue;
      const float u = t >= j ? src.get(row - j, a.off + c) : ld_elem(ring, (col % a.slots) * a.C + c);
      v += a.w[(int64_t)(a.taps - 1 - j) * a.C + c] * u;
    }
    if (a.T == 1) st_elem(ring, (int64_t)(slot % a.slots) * a.C + c, src.get(row, a.off + c));
    return v;
  };
  const float temp = query_temperature(max(slot - start, 0), a.coef, a.every);
  for (int it = tid; it < a.H * a.dkp; it += 256) {
    const int h = it / a.dkp, i = it % a.dkp;
    st_elem(q_out, (row * a.H + h) * a.dkp + i, i < a.dk ? convolved(a.q_off + (int64_t)h * a.dk + i) * temp : 0.f);
  }
  for (int it = tid; it < a.G * a.dkp; it += 256) {
    const int g = it / a.dkp, i = it % a.dkp;
    st_elem(kc, ((b * a.G + g) * a.S + slot) * a.dkp + i, i < a.dk ? convolved(a.k_off + (int64_t)g * a.dk + i) : 0.f);
  }
  for (int it = tid; it < a.G * a.dv; it += 256) vals[it] = convolved(a.v_off + it);
  __syncthreads();
  for (int g = tid >> 6; g < a.G; g += 4) {
    float s = 0.f;
    for (int i = tid & 63; i < a.dv; i += 64) s += vals[g * a.dv + i] * vals[g * a.dv + i];
    s = wave_sum(s);
    if ((tid & 63) == 0) vs[g] = a.value_norm ? 1.0f / sqrtf(s / (float)a.dv + a.eps) : 1.f;
  }
  __syncthreads();
  for (int it = tid; it < a.G * a.dvp; it += 256) {
    const int g = it / a.dvp, i = it % a.dvp;
    st_elem(vc, ((b * a.G + g) * a.S + slot) * a.dvp + i, i < a.dv ? vals[g * a.dv + i] * vs[g] : 0.f);
  }
}

// A group of `lanes` lanes (a power of two) owns one head over `run` tokens, a lane eight of its dimensions; the
// inputs of the tokens before stay in registers.
template <int TAPS, typename T>
__global__ __launch_bounds__(256) void conv_kvwrite_vec_kernel(const ConvKvArgs a, const RowSrc<T> src, T* q_out, T* kc, T* vc) {
  const int heads = a.H + 2 * a.G, runs = (int)((a.T + a.run - 1) / a.run), gl = threadIdx.x % a.lanes;
  const int64_t item = (int64_t)blockIdx.x * (256 / a.lanes) + threadIdx.x / a.lanes;
  if (item >= a.B * runs * heads) return;
  const int hd = (int)(item % heads), d0 = gl * 8;
  const int64_t b = item / heads / runs, t0 = item / heads % runs * a.run;
  const int kind = hd < a.H ? 0 : hd < a.H + a.G ? 1 : 2, g = kind == 0 ? hd : kind == 1 ? hd - a.H : hd - a.H - a.G;
  const int dim = kind == 2 ? a.dv : a.dk, pad = kind == 2 ? a.dvp : a.dkp;
  const bool real = d0 < dim;
  const int64_t c = (kind == 0 ? a.q_off : kind == 1 ? a.k_off : a.v_off) + (int64_t)g * dim + (real ? d0 : 0);
  const int col0 = *a.col_ptr, start = a.starts[b];
  T* ring = reinterpret_cast<T*>(a.ring) + b * a.slots * a.C;
  const RowSrc<T> rsrc{ring, nullptr, 1, 0, a.C};
  const RowSrc<float> wsrc{a.w, nullptr, 1, 0, a.C};
  float w[TAPS][8], u[TAPS][8];
#pragma unroll
  for (int k = 0; k < TAPS; ++k) get8(wsrc, k, c, w[k]);
  auto input = [&](int64_t t, float (&f)[8]) {
    const int64_t col = col0 + t;
    if (col < start) {
#pragma unroll
      for (int i = 0; i < 8; ++i) f[i] = 0.f;
    } else if (t >= 0) {
      get8(src, b * a.T + t, a.off + c, f);
    } else {
      get8(rsrc, col % a.slots, c, f);
    }
  };
#pragma unroll
  for (int k = 0; k + 1 < TAPS; ++k) input(t0 - (TAPS - 1) + k, u[k]);
  const int64_t t1 = min(a.T, t0 + a.run);
  for (int64_t t = t0; t < t1; ++t) {
    const int64_t row = b * a.T + t, slot = col0 + t;
    if (slot >= a.S) break;
    input(t, u[TAPS - 1]);
    float v[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      v[i] = 0.f;
#pragma unroll
      for (int k = 0; k < TAPS; ++k) v[i] += w[k][i] * u[k][i];
    }
    float f = 1.f;
    if (kind == 0) f = query_temperature(max((int)slot - start, 0), a.coef, a.every);
    if (kind == 2 && a.value_norm) {
      float s = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) s += v[i] * v[i];
      if (!real) s = 0.f;
      for (int o = a.lanes / 2; o > 0; o >>= 1) s += __shfl_xor(s, o, 64);
      f = 1.0f / sqrtf(s / (float)dim + a.eps);
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = real ? v[i] * f : 0.f;
    if (d0 < pad) {
      T* dst = kind == 0 ? q_out + (row * a.H + g) * a.dkp : kind == 1 ? kc + ((b * a.G + g) * a.S + slot) * a.dkp : vc + ((b * a.G + g) * a.S + slot) * a.dvp;
      put8(dst + d0, v);
    }
    if (a.T == 1 && real) put8(ring + (slot % a.slots) * a.C + c, u[TAPS - 1]);
#pragma unroll
    for (int k = 0; k + 1 < TAPS; ++k)
#pragma unroll
      for (int i = 0; i < 8; ++i) u[k][i] = u[k + 1][i];
  }
}
template <typename T>
int launch_conv_kv(hipStream_t st, ConvKvArgs a, const RowSrc<T>& src, T* q_out, T* kc, T* vc) {
  const bool vec = a.taps <= 4 && (a.dk | a.dv | a.dkp | a.dvp) % 8 == 0 && a.dkp <= 512 && a.dvp <= 512 && (a.off | a.C | a.q_off | a.k_off | a.v_off) % 8 == 0 &&
                   src.ld % 8 == 0 && src.plane % 8 == 0;
  if (!vec) {
    TNX_REQUIRE((int64_t)a.G * (a.dv + 1) <= 16000, "conv_kvwrite: values of one row above 16000");
    hipLaunchKernelGGL((conv_kvwrite_kernel<T>), dim3((unsigned)(a.B * a.T)), dim3(256), (size_t)a.G * (a.dv + 1) * 4, st, a, src, q_out, kc, vc);
    TNX_CHECK_LAUNCH("conv_kvwrite");
    return TNX_OK;
  }
  a.lanes = 1;
  while (a.lanes * 8 < (a.dkp > a.dvp ? a.dkp : a.dvp)) a.lanes *= 2;
  const int heads = a.H + 2 * a.G;
  a.run = 16;
  while (a.run > 1 && a.B * cdiv(a.T, a.run) * heads * a.lanes < 262144) a.run /= 2;
  const dim3 grid((unsigned)cdiv(a.B * cdiv(a.T, a.run) * heads, 256 / a.lanes));
  if (a.taps == 1) hipLaunchKernelGGL((conv_kvwrite_vec_kernel<1, T>), grid, dim3(256), 0, st, a, src, q_out, kc, vc);
  else if (a.taps == 2) hipLaunchKernelGGL((conv_kvwrite_vec_kernel<2, T>), grid, dim3(256), 0, st, a, src, q_out, kc, vc);
  else if (a.taps == 3) hipLaunchKernelGGL((conv_kvwrite_vec_kernel<3, T>), grid, dim3(256), 0, st, a, src, q_out, kc, vc);
  else hipLaunchKernelGGL((conv_kvwrite_vec_kernel<4, T>), grid, dim3(256), 0, st, a, src, q_out, kc, vc);
  TNX_CHECK_LAUNCH("conv_kvwrite");
  return TNX_OK;
}

__global__ __launch_bounds__(256) void soft_cap_kernel(float* z, int64_t n, float cap) {
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) z[i] = cap * tanhf(z[i] / cap);
}

// ---- rotation of the first rot_dims dimensions of q and k, cache write --------------------------
struct PartRopeArgs {
  int64_t T, S;
  int H, G, dk, dv, dkp, dvp, half;
  const float* inv_freq;
  const int32_t* starts;
  const int32_t* col_ptr;
  int64_t k_off, v_off;
};
constexpr int kMaxHalf = 256;

template <typename T>
__global__ __launch_bounds__(256) void part_rope_kernel(const PartRopeArgs a, const RowSrc<T> src, T* q_out, T* kc, T* vc) {
  __shared__ float sn[kMaxHalf], cs[kMaxHalf];
  const int64_t row = blockIdx.x, b = row / a.T, t = row % a.T;
  const int slot = *a.col_ptr + (int)t;
  if (slot >= a.S) return;                                    // (uniform; the host sizes the cache)
  const float pos = (float)max(slot - a.starts[b], 0);
  for (int i = threadIdx.x; i < a.half; i += 256) sincosf(pos * a.inv_freq[i], &sn[i], &cs[i]);
  __syncthreads();
  const int heads = a.H + a.G, hpt = a.dkp - a.half;           // one item per pair or lone dimension
  for (int it = threadIdx.x; it < heads * hpt; it += 256) {
    const int hd = it / hpt, i = it % hpt;
    const bool is_k = hd >= a.H;
    const int64_t base = is_k ? a.k_off + (int64_t)(hd - a.H) * a.dk : (int64_t)hd * a.dk;
    T* dst = is_k ? kc + ((b * a.G + (hd - a.H)) * a.S + slot) * a.dkp : q_out + (row * a.H + hd) * a.dkp;
    if (i < a.half) {
      const float u = src.get(row, base + i), v = src.get(row, base + i + a.half);
      st_elem(dst, i, u * cs[i] - v * sn[i]);
      st_elem(dst, i + a.half, v * cs[i] + u * sn[i]);
    } else {
      const int d = i + a.half;
      st_elem(dst, d, d < a.dk ? src.get(row, base + d) : 0.f);
    }
  }
  for (int it = threadIdx.x; it < a.G * a.dvp; it += 256) {
    const int g = it / a.dvp, d = it % a.dvp;
    st_elem(vc, ((b * a.G + g) * a.S + slot) * a.dvp + d, d < a.dv ? src.get(row, a.v_off + (int64_t)g * a.dv + d) : 0.f);
  }
}

// Heads, offsets and rotated halves in whole runs of eight: an item is eight dimensions (with their
// partners, where rotated) of one head; the items of a row are spread over gridDim.y work-groups.
template <typename T>
__global__ __launch_bounds__(256) void part_rope_vec_kernel(const PartRopeArgs a, const RowSrc<T> src, T* q_out, T* kc, T* vc) {
  __shared__ __align__(16) float sn[kMaxHalf], cs[kMaxHalf];
  const int64_t row = blockIdx.x, b = row / a.T, t = row % a.T;
  const int heads = a.H + a.G, hpt = (a.dkp - a.half) / 8, half8 = a.half / 8, vch = a.dvp / 8;
  const int n_rot = heads * hpt, n = n_rot + a.G * vch;
  const int first = blockIdx.y * 256 + threadIdx.x;
  const int slot = *a.col_ptr + (int)t;
  if (slot >= a.S) return;                                    // (uniform)
  const float pos = (float)max(slot - a.starts[b], 0);
  for (int i = threadIdx.x; i < a.half; i += 256) sincosf(pos * a.inv_freq[i], &sn[i], &cs[i]);
  __syncthreads();
  for (int it = first; it < n; it += 256 * gridDim.y) {
    float u[8];
    if (it >= n_rot) {
      const int g = (it - n_rot) / vch, d = ((it - n_rot) % vch) * 8;
      T* dst = vc + ((b * a.G + g) * a.S + slot) * a.dvp + d;
#pragma unroll
      for (int j = 0; j < 8; ++j) u[j] = 0.f;
      if (d < a.dv) get8(src, row, a.v_off + (int64_t)g * a.dv + d, u);
      put8(dst, u);
      continue;
    }
    const int hd = it / hpt, c = it % hpt;
    const bool is_k = hd >= a.H;
    const int64_t base = is_k ? a.k_off + (int64_t)(hd - a.H) * a.dk : (int64_t)hd * a.dk;
    T* dst = is_k ? kc + ((b * a.G + (hd - a.H)) * a.S + slot) * a.dkp : q_out + (row * a.H + hd) * a.dkp;
    if (c < half8) {
      float v[8], o1[8], o2[8];
      get8(src, row, base + c * 8, u);
      get8(src, row, base + a.half + c * 8, v);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float co = cs[c * 8 + j], si = sn[c * 8 + j];
        o1[j] = u[j] * co - v[j] * si;
        o2[j] = v[j] * co + u[j] * si;
      }
      put8(dst + c * 8, o1);
      put8(dst + a.half + c * 8, o2);
    } else {
      const int d = a.half + c * 8;
#pragma unroll
      for (int j = 0; j < 8; ++j) u[j] = 0.f;
      if (d < a.dk) get8(src, row, base + d, u);
      put8(dst + d, u);
    }
  }
}

// ---- RMS norm and a gate, in parts of a row: norm(o) . w . sigmoid(g), or norm(o . silu(g)) . w --------------
struct GatedNormArgs {
  int64_t W, o_ld, out_ld, g_off;
  float eps, w_offset;
  const float* w;
  const float* o;
  int out_frag, groups;
  int64_t w_len;           // weights repeat after so many columns
};
// the gate first, then norms over equal parts: any width that fits LDS
template <typename T>
__global__ __launch_bounds__(256) void gate_first_kernel(const GatedNormArgs a, const RowSrc<T> g, T* out) {
  extern __shared__ __align__(16) float v[];
  __shared__ float gs[1024];
  const int64_t row = blockIdx.x;
  const int per = (int)(a.W / a.groups), lane = threadIdx.x & 63;
  for (int64_t i = threadIdx.x; i < a.W; i += 256) v[i] = a.o[row * a.o_ld + i] * silu_f32(g.get(row, a.g_off + i));
  __syncthreads();
  for (int p = threadIdx.x >> 6; p < a.groups; p += 4) {
    float s = 0.f;
    for (int i = lane; i < per; i += 64) s += v[p * per + i] * v[p * per + i];
    s = wave_sum(s);
    if (lane == 0) gs[p] = 1.0f / sqrtf(s / (float)per + a.eps);
  }
  __syncthreads();
  for (int64_t i = threadIdx.x; i < a.W; i += 256)
    st_elem(out, a.out_frag ? frag_index(row, i, a.out_ld) : row * a.out_ld + i, v[i] * gs[i / per] * (a.w_offset + a.w[i]));
}
template <int MAXC, typename T>
__global__ __launch_bounds__(256) void gate_first_vec_kernel(const GatedNormArgs a, const RowSrc<T> g, T* out) {
  __shared__ float part[MAXC * 256], gs[MAXC * 256];
  const int64_t row = blockIdx.x;
  const int nch = (int)(a.W / 8), per = nch / a.groups;
  float o[MAXC][8], w[MAXC][8], gv[MAXC][8];
  const RowSrc<float> os{a.o, nullptr, 1, 0, a.o_ld}, wsrc{a.w, nullptr, 1, 0, 0};
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int64_t col = (int64_t)min(c * 256 + (int)threadIdx.x, nch - 1) * 8;
    get8(os, row, col, o[c]);
    get8(wsrc, 0, col, w[c]);
    get8(g, row, a.g_off + col, gv[c]);
  }
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    float q = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      o[c][j] *= silu_f32(gv[c][j]);
      q += o[c][j] * o[c][j];
    }
    part[c * 256 + threadIdx.x] = q;
  }
  part_scales(part, gs, a.groups, per, (float)(per * 8), a.eps);
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int ch = c * 256 + threadIdx.x;
    if (ch >= nch) continue;
    const float r = gs[ch / per];
#pragma unroll
    for (int j = 0; j < 8; ++j) o[c][j] = o[c][j] * r * (a.w_offset + w[c][j]);
    put8(out + (a.out_frag ? frag_index(row, (int64_t)ch * 8, a.out_ld) : row * a.out_ld + (int64_t)ch * 8), o[c]);
  }
}
template <typename T>
int launch_gate_first(hipStream_t st, int64_t M, const GatedNormArgs& a, const RowSrc<T>& g, T* out) {
  const dim3 grid((unsigned)M);
  const bool vec = a.W % 8 == 0 && a.W / a.groups % 8 == 0 && a.W <= 16384 && a.o_ld % 8 == 0 && g.ld % 8 == 0 && g.plane % 8 == 0 && a.g_off % 8 == 0 &&
                   a.out_ld % 8 == 0;
  if (!vec) {
    TNX_REQUIRE(a.W <= 15360 && a.groups <= 1024, "gated_norm: W=%lld in %d parts needs runs of eight", (long long)a.W, a.groups);
    hipLaunchKernelGGL((gate_first_kernel<T>), grid, dim3(256), (size_t)a.W * 4, st, a, g, out);
  } else if (a.W <= 2048) hipLaunchKernelGGL((gate_first_vec_kernel<1, T>), grid, dim3(256), 0, st, a, g, out);
  else if (a.W <= 4096) hipLaunchKernelGGL((gate_first_vec_kernel<2, T>), grid, dim3(256), 0, st, a, g, out);
  else if (a.W <= 8192) hipLaunchKernelGGL((gate_first_vec_kernel<4, T>), grid, dim3(256), 0, st, a, g, out);
  else hipLaunchKernelGGL((gate_first_vec_kernel<8, T>), grid, dim3(256), 0, st, a, g, out);
  TNX_CHECK_LAUNCH("gated_norm");
  return TNX_OK;
}
template <typename T>
__global__ __launch_bounds__(256) void gated_norm_kernel(const GatedNormArgs a, const RowSrc<T> g, T* out) {
  __shared__ float gs[1024];
  const int64_t row = blockIdx.x;
  const float* o = a.o + row * a.o_ld;
  const int per = (int)(a.W / a.groups), lane = threadIdx.x & 63;
  if (a.groups == 1) {
    float ss = 0.f;
    for (int64_t i = threadIdx.x; i < a.W; i += 256) ss += o[i] * o[i];
    ss = block_sum(ss, gs + 4);
    if (threadIdx.x == 0) gs[0] = 1.0f / sqrtf(ss / (float)a.W + a.eps);
  } else {
    for (int p = threadIdx.x >> 6; p < a.groups; p += 4) {
      float s = 0.f;
      for (int i = lane; i < per; i += 64) s += o[p * per + i] * o[p * per + i];
      s = wave_sum(s);
      if (lane == 0) gs[p] = 1.0f / sqrtf(s / (float)per + a.eps);
    }
  }
  __syncthreads();
  for (int64_t i = threadIdx.x; i < a.W; i += 256)
    st_elem(out, a.out_frag ? frag_index(row, i, a.out_ld) : row * a.out_ld + i,
            o[i] * gs[i / per] * (a.w_offset + a.w[i % a.w_len]) * (g.ld > 0 ? sigmoid_f32(g.get(row, a.g_off + i)) : 1.f));
}
// eight elements per thread and turn, everything requested ahead of the sum
template <int MAXC, bool PARTS, typename T>
__global__ __launch_bounds__(256) void gated_norm_vec_kernel(const GatedNormArgs a, const RowSrc<T> g, T* out) {
  __shared__ float red[4], part[PARTS ? MAXC * 256 : 1], gs[PARTS ? MAXC * 256 : 1];
  const int64_t row = blockIdx.x;
  const int nch = (int)(a.W / 8), per = nch / a.groups;
  float o[MAXC][8], w[MAXC][8], gv[MAXC][8];
  const RowSrc<float> os{a.o, nullptr, 1, 0, a.o_ld}, wsrc{a.w, nullptr, 1, 0, 0};
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int64_t col = (int64_t)min(c * 256 + (int)threadIdx.x, nch - 1) * 8;
    get8(os, row, col, o[c]);
    get8(wsrc, 0, PARTS ? col % a.w_len : col, w[c]);
    if (g.ld > 0) get8(g, row, a.g_off + col, gv[c]);   // (uniform)
  }
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    float q = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) q += o[c][j] * o[c][j];
    if constexpr (PARTS) part[c * 256 + threadIdx.x] = q;
    else if (c * 256 + (int)threadIdx.x < nch) ss += q;
  }
  float r = 1.f;
  if constexpr (PARTS) part_scales(part, gs, a.groups, per, (float)(per * 8), a.eps);
  else r = 1.0f / sqrtf(block_sum(ss, red) / (float)a.W + a.eps);
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int ch = c * 256 + threadIdx.x;
    if (ch >= nch) continue;
    if constexpr (PARTS) r = gs[ch / per];
#pragma unroll
    for (int j = 0; j < 8; ++j) o[c][j] = o[c][j] * r * (a.w_offset + w[c][j]) * (g.ld > 0 ? sigmoid_f32(gv[c][j]) : 1.f);
    put8(out + (a.out_frag ? frag_index(row, (int64_t)ch * 8, a.out_ld) : row * a.out_ld + (int64_t)ch * 8), o[c]);
  }
}
template <bool PARTS, typename T>
void launch_gated_norm_vec(hipStream_t st, int64_t M, const GatedNormArgs& a, const RowSrc<T>& g, T* out) {
  const dim3 grid((unsigned)M);
  if (a.W <= 2048) hipLaunchKernelGGL((gated_norm_vec_kernel<1, PARTS, T>), grid, dim3(256), 0, st, a, g, out);
  else if (a.W <= 4096) hipLaunchKernelGGL((gated_norm_vec_kernel<2, PARTS, T>), grid, dim3(256), 0, st, a, g, out);
  else if (a.W <= 8192) hipLaunchKernelGGL((gated_norm_vec_kernel<4, PARTS, T>), grid, dim3(256), 0, st, a, g, out);
  else hipLaunchKernelGGL((gated_norm_vec_kernel<8, PARTS, T>), grid, dim3(256), 0, st, a, g, out);
}
template <typename T>
void launch_gated_norm(hipStream_t st, int64_t M, const GatedNormArgs& a, const RowSrc<T>& g, T* out) {
  const bool vec = a.W % 8 == 0 && a.W / a.groups % 8 == 0 && a.W <= 16384 && a.o_ld % 8 == 0 && g.ld % 8 == 0 && g.plane % 8 == 0 && a.g_off % 8 == 0 &&
                   a.out_ld % 8 == 0;
  if (!vec) hipLaunchKernelGGL((gated_norm_kernel<T>), dim3((unsigned)M), dim3(256), 0, st, a, g, out);
  else if (a.groups > 1) launch_gated_norm_vec<true>(st, M, a, g, out);
  else launch_gated_norm_vec<false>(st, M, a, g, out);
}

// ---- gated unit on finished projections: out = act(y[:, :F]) * y[:, u_off : u_off + F] -----------
template <bool SILU, typename T>
__global__ __launch_bounds__(256) void act_mul_kernel(const T* y, int64_t ld, int64_t u_off, int64_t F, T* out, int64_t out_ld) {
  const int64_t row = blockIdx.y, i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= F) return;
  const float z = ld_elem(y, row * ld + i);
  st_elem(out, row * out_ld + i, (SILU ? silu_f32(z) : gelu_tanh_f32(z)) * ld_elem(y, row * ld + u_off + i));
}
template <bool SILU>
int launch_act_mul(hipStream_t st, int dtype, const void* y, int64_t ld, int64_t up_off, int64_t M, int64_t F, void* out, int64_t out_ld) {
  TNX_REQUIRE(y && out && M > 0 && F > 0 && ld >= up_off + F && out_ld >= F, "act_mul: null pointer or bad shape");
  TNX_REQUIRE(dtype == TNX_BF16 || dtype == TNX_F32, "act_mul: bad dtype %d", dtype);
  for (int64_t r0 = 0; r0 < M; r0 += 65535) {
    const int64_t n = M - r0 < 65535 ? M - r0 : 65535;
    const dim3 grid((unsigned)cdiv(F, 256), (unsigned)n);
    if (dtype == TNX_BF16)
      hipLaunchKernelGGL((act_mul_kernel<SILU, uint16_t>), grid, dim3(256), 0, st, (const uint16_t*)y + r0 * ld, ld, up_off, F,
                         (uint16_t*)out + r0 * out_ld, out_ld);
    else
      hipLaunchKernelGGL((act_mul_kernel<SILU, float>), grid, dim3(256), 0, st, (const float*)y + r0 * ld, ld, up_off, F,
                         (float*)out + r0 * out_ld, out_ld);
  }
  TNX_CHECK_LAUNCH("act_mul");
  return TNX_OK;
}

// ---- choice of experts: the k largest logits (first among equals), softmax over them ---------------
// One wave per token.  NaN logits rank below every number, so that k distinct experts are found whatever
// the logits hold; they leave as NaN weights.
// Up to 256 experts: every expert counts the ones ahead of it, which is its place among the chosen; more: one
// pass over the logits per choice.
constexpr int kRankExperts = 256;
__global__ __launch_bounds__(64) void route_softmax_kernel(const RowSrc<float> src, int E, int k, float* topk_w, int32_t* topk_id) {
  extern __shared__ __align__(16) float z[];   // logits [E], chosen logits [k]
  float* sel = z + E;
  const int64_t m = blockIdx.x;
  const int lane = threadIdx.x;
  const float ninf = -__builtin_inff();
  bool bad = false;
  for (int e = lane; e < E; e += 64) {
    const float v = src.get(m, e);
    bad |= v != v;
    z[e] = v == v ? fmaxf(v, -3.0e38f) : -3.0e38f;   // (a taken expert is -inf)
  }
  bad = __any(bad);
  __syncthreads();
  if (E <= kRankExperts) {   // (uniform)
    for (int e = lane; e < E; e += 64) {
      const float v = z[e];
      int ahead = 0;
      int o = 0;
      for (; o + 4 <= E; o += 4) {
        const f32x4 w = *reinterpret_cast<const f32x4*>(z + o);
#pragma unroll
        for (int i = 0; i < 4; ++i) ahead += w[i] > v || (w[i] == v && o + i < e);
      }
      for (; o < E; ++o) ahead += z[o] > v || (z[o] == v && o < e);
      if (ahead < k) {
        sel[ahead] = v;
        topk_id[m * k + ahead] = e;
      }
    }
    __syncthreads();
  }
  for (int j = 0; j < k && E > kRankExperts; ++j) {
    float best = ninf;
    int bi = 0x7fffffff;
    for (int e = lane; e < E; e += 64)
      if (z[e] > best) {
        best = z[e];
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
      sel[j] = best;
      topk_id[m * k + j] = bi;
      z[bi] = ninf;
    }
    __syncthreads();
  }
  float sum = 0.f;
  for (int j = lane; j < k; j += 64) sum += expf(sel[j] - sel[0]);
  sum = wave_sum(sum);
  for (int j = lane; j < k; j += 64) topk_w[m * k + j] = bad ? __builtin_nanf("") : expf(sel[j] - sel[0]) / sum;
}

// ---- statistics and the whole-vocabulary draw over finished fp32 logits -------------------------
struct LogitsArgs {
  int64_t M, V;
  const float* logits;
  float temperature;
  const int32_t* forbidden;
  int n_forbidden;
  const int32_t* targets;
  int32_t* best_id;
  float *best_logp, *target_logp, *lse, *entropy;
  uint32_t key0, key1;
  int variant;
  const int32_t* step_ptr;
  int32_t* draw_id;
  float* draw_logp;
};
struct Best {
  float v;
  int i;
};
__device__ __forceinline__ Best better(Best a, Best b) {   // larger value, then lower index
  return (b.v > a.v || (b.v == a.v && b.i < a.i)) ? b : a;
}
__device__ __forceinline__ Best block_best(Best v, Best* red) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v = better(v, Best{__shfl_xor(v.v, o, 64), __shfl_xor(v.i, o, 64)});
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  Best r = red[0];
  for (int w = 1; w < (int)(blockDim.x >> 6); ++w) r = better(r, red[w]);
  return r;
}
__global__ __launch_bounds__(256) void logits_stats_kernel(const LogitsArgs a) {
  __shared__ float red[4];
  __shared__ Best bred[4];
  const int64_t row = blockIdx.x;
  const float* l = a.logits + row * a.V;
  const float ninf = -__builtin_inff();
  auto value = [&](int64_t i) {
    for (int f = 0; f < a.n_forbidden; ++f)
      if (a.forbidden[f] == i) return ninf;
    return __fdiv_rn(l[i], a.temperature);
  };
  uint32_t ks0 = 0u, ks1 = 0u;
  if (a.draw_id) {
    ks1 = (uint32_t)(*a.step_ptr);
    threefry2x32(a.key0, a.key1, ks0, ks1);
  }
  Best top{ninf, 0x7fffffff}, drawn{ninf, 0x7fffffff};
  for (int64_t i = threadIdx.x; i < a.V; i += 256) {
    const float v = value(i);
    top = better(top, Best{v, (int)i});
    if (a.draw_id && v != ninf)
      drawn = better(drawn, Best{v + gumbel_from_bits(random_bits(ks0, ks1, (uint64_t)row * (uint64_t)a.V + (uint64_t)i,
                                                                   (uint64_t)a.M * (uint64_t)a.V, a.variant)), (int)i});
  }
  top = block_best(top, bred);
  if (a.draw_id) drawn = block_best(drawn, bred);
  float se = 0.f, we = 0.f;
  for (int64_t i = threadIdx.x; i < a.V; i += 256) {
    const float v = value(i);
    if (v == ninf) continue;
    const float e = expf(v - top.v);
    se += e;
    we += e * v;
  }
  se = block_sum(se, red);
  we = block_sum(we, red);
  if (threadIdx.x == 0) {
    const float lse = top.v + logf(se);
    if (a.best_id) a.best_id[row] = top.i;
    if (a.best_logp) a.best_logp[row] = top.v - lse;
    if (a.target_logp) {
      const int t = a.targets[row];
      a.target_logp[row] = (t >= 0 && t < a.V ? value(t) : ninf) - lse;
    }
    if (a.lse) a.lse[row] = lse;
    if (a.entropy) a.entropy[row] = lse - we / se;
    if (a.draw_id) {
      a.draw_id[row] = drawn.i;
      if (a.draw_logp) a.draw_logp[row] = (drawn.i < a.V ? value(drawn.i) : ninf) - lse;
    }
  }
}

template <typename T>
RowSrc<T> row_src(const tnx_rows_src& s) {
  return RowSrc<T>{reinterpret_cast<const T*>(s.y), s.ws, s.split_k, s.plane, s.ld};
}

}  // namespace

extern "C" int tnx_embed_rows(void* stream, int dtype, const void* table, int64_t V, int64_t D, const int32_t* ids,
                              int64_t ids_ld, const int32_t* col_ptr, int64_t B, int64_t T, float scale, float* x, void* cat,
                              int64_t cat_ld, int64_t cat_off, int cat_frag, const void* pos, int64_t n_pos,
                              const int32_t* starts) {
  TNX_REQUIRE(table && ids && x, "embed_rows: null pointer");
  TNX_REQUIRE(V > 0 && D > 0 && B > 0 && T > 0, "embed_rows: bad shape");
  TNX_REQUIRE(!cat || (cat_ld >= cat_off + D && cat_off % D == 0), "embed_rows: the second copy does not fit its rows");
  TNX_REQUIRE(!pos || (n_pos > 0 && starts), "embed_rows: learned positions need their number and the first columns");
  TNX_REQUIRE(dtype == TNX_BF16 || dtype == TNX_F32, "embed_rows: bad dtype %d", dtype);
  if (dtype == TNX_BF16)
    hipLaunchKernelGGL(embed_rows_kernel<uint16_t>, dim3((unsigned)(B * T)), dim3(256), 0, as_stream(stream), (const uint16_t*)table,
                       V, D, ids, ids_ld, col_ptr, T, scale, x, (uint16_t*)cat, cat_ld, cat_off, cat_frag, (const uint16_t*)pos, n_pos, starts);
  else
    hipLaunchKernelGGL(embed_rows_kernel<float>, dim3((unsigned)(B * T)), dim3(256), 0, as_stream(stream), (const float*)table, V, D,
                       ids, ids_ld, col_ptr, T, scale, x, (float*)cat, cat_ld, cat_off, cat_frag, (const float*)pos, n_pos, starts);
  TNX_CHECK_LAUNCH("embed_rows");
  return TNX_OK;
}

extern "C" int tnx_residual_norm(void* stream, const tnx_residual_norm_desc* d) {
  TNX_REQUIRE(d, "residual_norm: null descriptor");
  TNX_REQUIRE(d->M > 0 && d->D > 0 && d->D <= 16384, "residual_norm: D=%lld out of range (1..16384)", (long long)d->D);
  TNX_REQUIRE(d->x && d->out && d->out_ld >= d->D, "residual_norm: null pointer or short output rows");
  TNX_REQUIRE(d->mode >= 0 && d->mode <= 3, "residual_norm: bad mode %d", d->mode);
  const bool arrives = d->mode == 1 || d->mode == 2;
  TNX_REQUIRE(!arrives || d->y.y || d->y.ws, "residual_norm: no incoming rows");
  TNX_REQUIRE((d->mode != 1 && d->mode != 3) || d->w_post, "residual_norm: null post-norm weight");
  const int groups = d->groups < 1 ? 1 : d->groups;
  TNX_REQUIRE(d->D % groups == 0, "residual_norm: D=%lld does not divide into %d parts", (long long)d->D, groups);
  TNX_REQUIRE(!d->route_w || (d->route_k > 0 && arrives && d->y.y && d->y.split_k <= 1), "residual_norm: routed rows are finished, and need their number per row");
  TNX_REQUIRE(!d->shift || (!d->w_next && d->before && d->starts && d->col_ptr && d->B > 0 && d->T > 0 && d->B * d->T == d->M),
              "residual_norm: a shift needs the rows before, their columns and no next norm");
  TNX_REQUIRE(!d->shift || d->T == 1 || (d->x_out && d->x_out != d->x), "residual_norm: a shift over several tokens needs a second buffer");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "residual_norm: bad dtype %d", d->dtype);
  if (d->center || (d->mult != 0.f && d->mult != 1.f) || d->extra.ld > 0 || d->hist) return tnx_internal_layer_step(as_stream(stream), d);
  ResNormArgs a;
  a.M = d->M; a.D = d->D; a.eps = d->eps; a.w_offset = d->w_offset; a.y = d->y.y; a.ws = d->y.ws;
  a.split = d->y.split_k < 1 ? 1 : d->y.split_k; a.plane = d->y.plane; a.y_ld = arrives ? d->y.ld : 8; a.mode = d->mode;
  a.w_post = d->w_post; a.x = d->x; a.w_next = d->w_next; a.out = d->out; a.out_ld = d->out_ld; a.out_frag = d->out_frag;
  if (!arrives) a.plane = 0;
  a.groups = groups; a.x_out = d->x_out ? d->x_out : d->x; a.route_w = d->route_w; a.route_k = d->route_k; a.shift = d->shift;
  a.before = d->before; a.starts = d->starts; a.col_ptr = d->col_ptr; a.B = d->shift ? d->B : 1; a.T = d->shift ? d->T : d->M;
  if (groups > 1 || d->mode == 3 || d->route_w || d->shift || a.x_out != a.x) {
    const int rc = d->dtype == TNX_BF16 ? launch_resnorm_rows<uint16_t>(as_stream(stream), a) : launch_resnorm_rows<float>(as_stream(stream), a);
    if (rc) return rc;
    TNX_CHECK_LAUNCH("residual_norm");
    return TNX_OK;
  }
  if (d->dtype == TNX_BF16) launch_resnorm<uint16_t>(as_stream(stream), a);
  else launch_resnorm<float>(as_stream(stream), a);
  TNX_CHECK_LAUNCH("residual_norm");
  return TNX_OK;
}

extern "C" int tnx_parallel_step(void* stream, const tnx_parallel_step_desc* d) {
  TNX_REQUIRE(d, "parallel_step: null descriptor");
  TNX_REQUIRE(d->M > 0 && d->D > 0 && d->B > 0 && d->T > 0 && d->B * d->T == d->M && d->M < (int64_t)1 << 31, "parallel_step: bad shape");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "parallel_step: bad dtype %d", d->dtype);
  TNX_REQUIRE(d->n_in >= 0 && d->n_in <= 3, "parallel_step: %d incoming rows, at most three", d->n_in);
  TNX_REQUIRE(d->x && d->w_next && d->out1 && d->out_ld >= d->D, "parallel_step: null pointer or short output rows");
  TNX_REQUIRE(d->x_out || (d->n_in == 0 && !d->add), "parallel_step: the new residual needs a buffer");
  TNX_REQUIRE(!d->out2 || (d->conv1 && d->conv2), "parallel_step: a second output needs both convolutions");
  const int taps = d->conv1 ? d->taps : 1;
  if (d->conv1) {
    TNX_REQUIRE(taps >= 1 && taps <= 4096 && d->starts && d->col_ptr, "parallel_step: the convolutions need taps and columns");
    TNX_REQUIRE(taps == 1 || (d->ring && d->slots >= taps - 1 && (d->T == 1 || (d->tail && (!d->x_out || d->x_out != d->x)))),
                "parallel_step: the convolutions need a ring and, over several tokens, a tail and a second residual buffer");
  }
  ParallelArgs a;
  memset(&a, 0, sizeof(a));
  a.D = d->D; a.B = d->B; a.T = d->T; a.eps = d->eps; a.mult = d->mult; a.n_in = d->n_in;
  for (int p = 0; p < d->n_in; ++p) {
    TNX_REQUIRE(src_given(d->y[p]) && d->y[p].ld >= d->D, "parallel_step: incoming rows %d are missing", p);
    a.y[p] = d->y[p].y; a.ws[p] = d->y[p].ws; a.split[p] = d->y[p].split_k < 1 ? 1 : d->y[p].split_k; a.plane[p] = a.split[p] > 1 ? d->y[p].plane : 0;
    a.y_ld[p] = d->y[p].ld; a.w_post[p] = d->w_post[p]; a.y_scale[p] = d->y_scale[p];
  }
  a.x = d->x; a.x_out = d->x_out; a.add = d->add; a.w_next = d->w_next; a.taps = taps; a.slots = d->slots; a.conv1 = d->conv1;
  a.conv2 = d->out2 ? d->conv2 : nullptr; a.out1 = d->out1; a.out2 = d->out2; a.out_ld = d->out_ld; a.out_frag = d->out_frag;
  a.ring = d->ring; a.tail = d->tail; a.starts = d->starts; a.col_ptr = d->col_ptr;
  return d->dtype == TNX_BF16 ? launch_parallel<uint16_t>(as_stream(stream), a) : launch_parallel<float>(as_stream(stream), a);
}

extern "C" int tnx_conv_kvwrite(void* stream, const tnx_conv_kvwrite_desc* d) {
  TNX_REQUIRE(d, "conv_kvwrite: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->T > 0 && d->S > 0 && d->H > 0 && d->G > 0 && d->H % d->G == 0 && d->B * d->T < (int64_t)1 << 31, "conv_kvwrite: bad shape");
  TNX_REQUIRE(d->dk > 0 && d->dv > 0 && d->dkp >= d->dk && d->dvp >= d->dv, "conv_kvwrite: bad head sizes");
  TNX_REQUIRE(d->taps >= 1 && d->taps <= 4096 && d->slots >= 1 && d->slots >= (d->T == 1 ? d->taps : d->taps - 1), "conv_kvwrite: the ring is shorter than the taps");
  TNX_REQUIRE(d->off >= 0 && d->q_off >= 0 && d->k_off >= 0 && d->v_off >= 0 && d->q_off + (int64_t)d->H * d->dk <= d->C && d->k_off + (int64_t)d->G * d->dk <= d->C &&
                  d->v_off + (int64_t)d->G * d->dv <= d->C,
              "conv_kvwrite: heads outside the channels");
  TNX_REQUIRE(src_given(d->y) && d->w && d->ring && d->starts && d->col_ptr && d->q_out && d->kcache && d->vcache && d->temp_every > 0.f, "conv_kvwrite: null pointer");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "conv_kvwrite: bad dtype %d", d->dtype);
  ConvKvArgs a;
  memset(&a, 0, sizeof(a));
  a.B = d->B; a.T = d->T; a.S = d->S; a.H = d->H; a.G = d->G; a.dk = d->dk; a.dv = d->dv; a.dkp = d->dkp; a.dvp = d->dvp; a.taps = d->taps; a.slots = d->slots;
  a.coef = d->temp_coef; a.every = d->temp_every; a.eps = d->eps; a.value_norm = d->value_norm; a.off = d->off; a.C = d->C; a.q_off = d->q_off;
  a.k_off = d->k_off; a.v_off = d->v_off; a.w = d->w; a.ring = d->ring; a.starts = d->starts; a.col_ptr = d->col_ptr;
  if (d->dtype == TNX_BF16)
    return launch_conv_kv(as_stream(stream), a, row_src<uint16_t>(d->y), (uint16_t*)d->q_out, (uint16_t*)d->kcache, (uint16_t*)d->vcache);
  return launch_conv_kv(as_stream(stream), a, row_src<float>(d->y), (float*)d->q_out, (float*)d->kcache, (float*)d->vcache);
}

extern "C" int tnx_soft_cap(void* stream, float* z, int64_t n, float cap) {
  TNX_REQUIRE(z && n > 0 && cap > 0.f, "soft_cap: null pointer or bad shape");
  const int64_t blocks = cdiv(n, 1024);
  hipLaunchKernelGGL(soft_cap_kernel, dim3((unsigned)(blocks < 65535 ? blocks : 65535)), dim3(256), 0, as_stream(stream), z, n, cap);
  TNX_CHECK_LAUNCH("soft_cap");
  return TNX_OK;
}

extern "C" int tnx_part_rope_kvwrite(void* stream, const tnx_part_rope_desc* d) {
  TNX_REQUIRE(d, "part_rope: null descriptor");
  TNX_REQUIRE(d->B > 0 && d->T > 0 && d->S > 0 && d->H > 0 && d->G > 0 && d->H % d->G == 0, "part_rope: bad shape");
  TNX_REQUIRE(d->dk > 0 && d->dv > 0 && d->dkp >= d->dk && d->dvp >= d->dv, "part_rope: bad head sizes");
  TNX_REQUIRE(d->rot_dims >= 0 && d->rot_dims % 2 == 0 && d->rot_dims <= d->dk && d->rot_dims / 2 <= kMaxHalf,
              "part_rope: rot_dims=%d must be even, at most the head size and at most 512", d->rot_dims);
  TNX_REQUIRE(src_given(d->y) && d->starts && d->col_ptr && d->q_out && d->kcache && d->vcache && (d->rot_dims == 0 || d->inv_freq),
              "part_rope: null pointer");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "part_rope: bad dtype %d", d->dtype);
  PartRopeArgs a;
  a.T = d->T; a.S = d->S; a.H = d->H; a.G = d->G; a.dk = d->dk; a.dv = d->dv; a.dkp = d->dkp; a.dvp = d->dvp;
  a.half = d->rot_dims / 2; a.inv_freq = d->inv_freq; a.starts = d->starts; a.col_ptr = d->col_ptr;
  a.k_off = d->k_off; a.v_off = d->v_off;
  const dim3 grid((unsigned)(d->B * d->T));
  hipStream_t st = as_stream(stream);
  const bool vec = d->dk % 8 == 0 && d->dv % 8 == 0 && d->dkp % 8 == 0 && d->dvp % 8 == 0 && a.half % 8 == 0 && d->k_off % 8 == 0 &&
                   d->v_off % 8 == 0 && d->y.ld % 8 == 0 && d->y.plane % 8 == 0;
  const bool bf = d->dtype == TNX_BF16;
  uint16_t *q16 = (uint16_t*)d->q_out, *k16 = (uint16_t*)d->kcache, *v16 = (uint16_t*)d->vcache;
  float *q32 = (float*)d->q_out, *k32 = (float*)d->kcache, *v32 = (float*)d->vcache;
  if (vec) {
    // few rows: one item per thread; many rows fill the device by themselves
    const int items = (d->H + d->G) * ((d->dkp - a.half) / 8) + d->G * (d->dvp / 8);
    const unsigned ny = d->B * d->T >= 1024 ? 1 : (unsigned)cdiv(items, 256);
    const dim3 g2((unsigned)(d->B * d->T), ny);
    if (bf) hipLaunchKernelGGL(part_rope_vec_kernel<uint16_t>, g2, dim3(256), 0, st, a, row_src<uint16_t>(d->y), q16, k16, v16);
    else hipLaunchKernelGGL(part_rope_vec_kernel<float>, g2, dim3(256), 0, st, a, row_src<float>(d->y), q32, k32, v32);
  } else if (bf) {
    hipLaunchKernelGGL(part_rope_kernel<uint16_t>, grid, dim3(256), 0, st, a, row_src<uint16_t>(d->y), q16, k16, v16);
  } else {
    hipLaunchKernelGGL(part_rope_kernel<float>, grid, dim3(256), 0, st, a, row_src<float>(d->y), q32, k32, v32);
  }
  TNX_CHECK_LAUNCH("part_rope");
  return TNX_OK;
}

extern "C" int tnx_gated_norm(void* stream, const tnx_gated_norm_desc* d) {
  TNX_REQUIRE(d, "gated_norm: null descriptor");
  TNX_REQUIRE(d->M > 0 && d->W > 0 && d->o && d->o_ld >= d->W && (src_given(d->g) || (d->g.ld == 0 && !d->gate_first)) && d->w && d->out && d->out_ld >= d->W,
              "gated_norm: null pointer or bad shape");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "gated_norm: bad dtype %d", d->dtype);
  GatedNormArgs a;
  a.W = d->W; a.o_ld = d->o_ld; a.out_ld = d->out_ld; a.g_off = d->g_off; a.eps = d->eps; a.w_offset = d->w_offset;
  a.w = d->w; a.o = d->o; a.out_frag = d->out_frag; a.groups = d->groups < 1 ? 1 : d->groups;
  a.w_len = d->shared_w ? d->W / a.groups : d->W;
  TNX_REQUIRE(!d->shared_w || !d->gate_first, "gated_norm: shared weights go with the gate behind the norm");
  TNX_REQUIRE(d->W % a.groups == 0 && a.groups <= 1024, "gated_norm: the row does not divide into %d parts, or into more than 1024", a.groups);
  if (d->gate_first)
    return d->dtype == TNX_BF16 ? launch_gate_first(as_stream(stream), d->M, a, row_src<uint16_t>(d->g), (uint16_t*)d->out)
                                : launch_gate_first(as_stream(stream), d->M, a, row_src<float>(d->g), (float*)d->out);
  if (d->dtype == TNX_BF16) launch_gated_norm(as_stream(stream), d->M, a, row_src<uint16_t>(d->g), (uint16_t*)d->out);
  else launch_gated_norm(as_stream(stream), d->M, a, row_src<float>(d->g), (float*)d->out);
  TNX_CHECK_LAUNCH("gated_norm");
  return TNX_OK;
}

extern "C" int tnx_gelu_mul(void* stream, int dtype, const void* y, int64_t ld, int64_t up_off, int64_t M, int64_t F, void* out,
                            int64_t out_ld) {
  return launch_act_mul<false>(as_stream(stream), dtype, y, ld, up_off, M, F, out, out_ld);
}

extern "C" int tnx_silu_mul(void* stream, int dtype, const void* y, int64_t ld, int64_t up_off, int64_t M, int64_t F, void* out,
                            int64_t out_ld) {
  return launch_act_mul<true>(as_stream(stream), dtype, y, ld, up_off, M, F, out, out_ld);
}

extern "C" int tnx_route_softmax(void* stream, const tnx_rows_src* z, int64_t M, int E, int k, float* topk_w, int32_t* topk_id) {
  TNX_REQUIRE(z && src_given(*z) && topk_w && topk_id, "route_softmax: null pointer");
  TNX_REQUIRE(M > 0 && M < ((int64_t)1 << 31) && E > 0 && E <= 4096 && k > 0 && k <= E && z->ld >= E, "route_softmax: bad shape E=%d k=%d", E, k);
  hipLaunchKernelGGL(route_softmax_kernel, dim3((unsigned)M), dim3(64), (size_t)(E + k) * 4, as_stream(stream), row_src<float>(*z), E, k,
                     topk_w, topk_id);
  TNX_CHECK_LAUNCH("route_softmax");
  return TNX_OK;
}

extern "C" int tnx_logits_stats(void* stream, const tnx_logits_desc* d) {
  TNX_REQUIRE(d && d->logits && d->M > 0 && d->V > 0 && d->V < (1LL << 31), "logits_stats: null pointer or bad shape");
  TNX_REQUIRE(!d->target_logp || d->targets, "logits_stats: target log-probabilities need targets");
  LogitsArgs a;
  memset(&a, 0, sizeof(a));
  a.M = d->M; a.V = d->V; a.logits = d->logits; a.temperature = d->temperature == 0.f ? 1.0f : d->temperature;
  a.forbidden = d->forbidden; a.n_forbidden = d->forbidden ? d->n_forbidden : 0; a.targets = d->targets;
  a.best_id = d->best_id; a.best_logp = d->best_logp; a.target_logp = d->target_logp; a.lse = d->lse; a.entropy = d->entropy;
  if (d->draw_id) {
    TNX_REQUIRE(d->draw_step_ptr && (d->draw_rng_variant == 0 || d->draw_rng_variant == 1) && d->temperature > 0.f,
                "logits_stats: the draw needs a step pointer, a known rng_variant and a positive temperature");
    a.key0 = d->draw_key0; a.key1 = d->draw_key1; a.variant = d->draw_rng_variant; a.step_ptr = d->draw_step_ptr;
    a.draw_id = d->draw_id; a.draw_logp = d->draw_logp;
  }
  hipLaunchKernelGGL(logits_stats_kernel, dim3((unsigned)d->M), dim3(256), 0, as_stream(stream), a);
  TNX_CHECK_LAUNCH("logits_stats");
  return TNX_OK;
}
