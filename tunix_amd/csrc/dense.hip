// Linears with dense weights (bf16 or fp32) for decoders whose weights are not quantised.
//
// bf16: the weights live in HBM once, in the fragment order of tnx_dense_expand.  Calls with many
// rows take the 128 x 256 kernel of qgemm_wide.h; calls with few rows take dense_rows_kernel below,
// which streams the same copy.  fp32: a plain tiled kernel in true 32-bit arithmetic.
#include <string.h>

#include <mutex>

#include "decoder.h"

int tnx_internal_wide_dense(hipStream_t st, int64_t M, int64_t K, int64_t N, const uint16_t* x, const uint16_t* w,
                            int epilogue, void* y, int64_t ldy);

namespace {

struct DenseArgs {
  int64_t M, K, N, ldy, ldx;
  const uint16_t* x;
  const uint16_t* w;
  void* y;
  float* ws;
  int epilogue, x_frag, y_frag, split_k;
};

typedef float f32x16 __attribute__((ext_vector_type(16)));
__device__ __forceinline__ f32x16 mfma32(u32x4 a, u32x4 b, f32x16 c) {
  // D[32x32] += A[32x16] * B[16x32]; lane l holds A row l%32 / B column l%32, k = 8*(l/32)..+7;
  // D: column l%32, rows 8*(r/4) + 4*(l/32) + r%4 for register r.
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}

constexpr int kDenseKT = 128;   // k-tile of the fragment layout: eight 16-deep slabs

// A work-group of four waves owns 32 * RT rows x 64 columns (two 32-column groups); its waves take
// the k-tiles of the work-group's k range in turn and meet through LDS at the end.  A slab of a
// column group is one 16-byte load per lane (1 KB per wave, contiguous), eight slabs ahead of
// their use in a register ring; activations in fragment order come the same way from L2.
// Products are formed transposed (weights as the MFMA's A operand): a lane owns runs of four
// consecutive columns of one row.
template <int RT>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, RT == 4 ? 1 : RT == 2 ? 2 : 4)))
void dense_rows_kernel(const DenseArgs a) {
  constexpr int CG = 2, XD = 4;   // column groups; slabs of activations in flight
  __shared__ __align__(16) float red[4][CG * 16 * 64];
  const int tid = threadIdx.x, lane = tid & 63, l32 = lane & 31, lh = lane >> 5;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int64_t m0 = (int64_t)blockIdx.y * (32 * RT);
  const int c64 = blockIdx.x, z = blockIdx.z;
  const int ktiles = (int)(a.K / kDenseKT);
  const int per = (ktiles + a.split_k - 1) / a.split_k;
  const int kt0 = z * per, kt1 = min(ktiles, kt0 + per);

  f32x16 acc[RT][CG];
#pragma unroll
  for (int rt = 0; rt < RT; ++rt)
#pragma unroll
    for (int cg = 0; cg < CG; ++cg)
#pragma unroll
      for (int i = 0; i < 16; ++i) acc[rt][cg][i] = 0.f;

  // [N/256][K/128][4 waves][2 groups][8 slabs][64 lanes] x 16 B; this work-group is wave c64 % 4 of tile c64 / 4
  const u32x4* wb = reinterpret_cast<const u32x4*>(a.w) + ((int64_t)(c64 >> 2) * ktiles * 8 + (c64 & 3) * 2) * 512 + lane;
  const u32x4* xf = reinterpret_cast<const u32x4*>(a.x);
  const int64_t kslabs = a.K / 16;
  const int64_t xrow0 = min(m0 + l32, a.M - 1);
  auto load_x = [&](int slab, int rt) -> u32x4 {
    if (a.x_frag) return xf[((m0 / 32 + rt) * kslabs + slab) * 64 + lane];
    const int64_t row = min(xrow0 + rt * 32, a.M - 1);
    return *reinterpret_cast<const u32x4*>(a.x + row * a.ldx + slab * 16 + lh * 8);
  };
  // the last row blocks of a partly filled tile: their fragments are in the (padded) buffer too
  u32x4 wr[8][CG];
  auto load_w = [&](int kt, int u) {
#pragma unroll
    for (int cg = 0; cg < CG; ++cg) wr[u][cg] = wb[((int64_t)kt * 8 + cg) * 512 + u * 64];
  };
  int kt = kt0 + wave;
  if (kt < kt1) {
#pragma unroll
    for (int u = 0; u < 8; ++u) load_w(kt, u);
    u32x4 xr[XD][RT];
#pragma unroll
    for (int u = 0; u < XD - 1; ++u)
#pragma unroll
      for (int rt = 0; rt < RT; ++rt) xr[u][rt] = load_x(kt * 8 + u, rt);
    for (; kt < kt1; kt += 4) {
      const int ktn = min(kt + 4, kt1 - 1);   // (past the end: a valid tile, loaded and not used)
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const int n = u + XD - 1, nslab = n < 8 ? kt * 8 + n : ktn * 8 + n - 8;
#pragma unroll
        for (int rt = 0; rt < RT; ++rt) xr[n % XD][rt] = load_x(nslab, rt);
#pragma unroll
        for (int cg = 0; cg < CG; ++cg)
#pragma unroll
          for (int rt = 0; rt < RT; ++rt) acc[rt][cg] = mfma32(wr[u][cg], xr[u % XD][rt], acc[rt][cg]);
        load_w(ktn, u);
      }
    }
  }

  // the four waves' parts meet, one row tile at a time; wave w then owns one quarter of the tile
  const bool mul = a.epilogue == TNX_EPI_GELU_MUL;
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) {
    __syncthreads();
#pragma unroll
    for (int cg = 0; cg < CG; ++cg)
#pragma unroll
      for (int i = 0; i < 4; ++i)
        *reinterpret_cast<f32x4*>(&red[wave][((cg * 4 + i) * 64 + lane) * 4]) =
            f32x4{acc[rt][cg][4 * i], acc[rt][cg][4 * i + 1], acc[rt][cg][4 * i + 2], acc[rt][cg][4 * i + 3]};
    __syncthreads();
    auto total = [&](int cg, int b) -> f32x4 {
      f32x4 s = *reinterpret_cast<const f32x4*>(&red[0][((cg * 4 + b) * 64 + lane) * 4]);
#pragma unroll
      for (int w = 1; w < 4; ++w) s += *reinterpret_cast<const f32x4*>(&red[w][((cg * 4 + b) * 64 + lane) * 4]);
      return s;
    };
    const int64_t row = m0 + rt * 32 + l32;
    if (row >= a.M) continue;
    if (mul) {
      // a 32-column group is [16 gate | 16 up]: quarters b and b + 2 pair up
      const int cg = wave >> 1, b = wave & 1;
      const f32x4 g = total(cg, b), u = total(cg, b + 2);
      const int64_t col = (int64_t)(c64 * 2 + cg) * 16 + 8 * b + 4 * lh;
      if (col >= a.N / 2) continue;
      const u32x2 pk = {pack2bf(gelu_tanh_f32(g[0]) * u[0], gelu_tanh_f32(g[1]) * u[1]),
                        pack2bf(gelu_tanh_f32(g[2]) * u[2], gelu_tanh_f32(g[3]) * u[3])};
      uint16_t* y = reinterpret_cast<uint16_t*>(a.y);
      *reinterpret_cast<u32x2*>(y + (a.y_frag ? frag_index(row, col, a.ldy) : row * a.ldy + col)) = pk;
      continue;
    }
#pragma unroll
    for (int cg = 0; cg < CG; ++cg) {
      const f32x4 v = total(cg, wave);
      const int64_t col = (int64_t)(c64 * 2 + cg) * 32 + 8 * wave + 4 * lh;
      if (a.epilogue == TNX_EPI_F32 || a.split_k > 1) {
        float* y = a.split_k > 1 ? a.ws + (int64_t)z * a.M * a.ldy : reinterpret_cast<float*>(a.y);
        y += row * a.ldy + col;
        if (col + 4 <= a.N && (a.ldy & 3) == 0) {
          *reinterpret_cast<f32x4*>(y) = v;
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (col + e < a.N) y[e] = v[e];
        }
      } else if (col < a.N) {   // bf16: N is a multiple of 16
        uint16_t* y = reinterpret_cast<uint16_t*>(a.y);
        *reinterpret_cast<u32x2*>(y + (a.y_frag ? frag_index(row, col, a.ldy) : row * a.ldy + col)) =
            u32x2{pack2bf(v[0], v[1]), pack2bf(v[2], v[3])};
      }
    }
  }
}

// fp32: 64 x 64 tile, 256 threads, 4 x 4 outputs each; K a multiple of 16
__global__ __launch_bounds__(256) void dense_f32_kernel(const float* x, int64_t ldx, const float* w, float* y,
                                                        int64_t ldy, int64_t M, int64_t K, int64_t N) {
  __shared__ float xs[16][68], wsh[16][68];
  const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
  const int64_t m0 = (int64_t)blockIdx.y * 64, n0 = (int64_t)blockIdx.x * 64;
  const int lr = tid >> 2, lk = (tid & 3) * 4;
  float acc[4][4] = {};
  for (int64_t k0 = 0; k0 < K; k0 += 16) {
    f32x4 xv = f32x4{0.f, 0.f, 0.f, 0.f}, wv = xv;
    if (m0 + lr < M) xv = *reinterpret_cast<const f32x4*>(x + (m0 + lr) * ldx + k0 + lk);
    if (n0 + lr < N) wv = *reinterpret_cast<const f32x4*>(w + (n0 + lr) * K + k0 + lk);
    __syncthreads();
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      xs[lk + e][lr] = xv[e];
      wsh[lk + e][lr] = wv[e];
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 16; ++k) {
      const f32x4 av = *reinterpret_cast<const f32x4*>(&xs[k][ty * 4]);
      const f32x4 bv = *reinterpret_cast<const f32x4*>(&wsh[k][tx * 4]);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] += av[i] * bv[j];
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (m0 + ty * 4 + i < M && n0 + tx * 4 + j < N) y[(m0 + ty * 4 + i) * ldy + n0 + tx * 4 + j] = acc[i][j];
}

}  // namespace

extern "C" int tnx_dense_linear(void* stream, const tnx_dense_desc* d) {
  TNX_REQUIRE(d, "dense_linear: null descriptor");
  TNX_REQUIRE(d->M > 0 && d->K > 0 && d->N > 0, "dense_linear: M, K, N must be positive");
  TNX_REQUIRE(d->x && d->w && (d->y || d->split_k > 1), "dense_linear: null pointer");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "dense_linear: bad dtype %d", d->dtype);
  hipStream_t st = as_stream(stream);
  if (d->dtype == TNX_F32) {
    TNX_REQUIRE(d->K % 16 == 0 && d->ldx % 4 == 0 && d->ldx >= d->K && d->ldy >= d->N,
                "dense_linear: fp32 needs K %% 16 == 0 and row strides that hold the rows");
    TNX_REQUIRE((d->epilogue == TNX_EPI_STORE || d->epilogue == TNX_EPI_F32) && d->split_k <= 1 && !d->x_frag && !d->y_frag,
                "dense_linear: fp32 stores row-major results only");
    TNX_REQUIRE(cdiv(d->M, 64) <= 65535, "dense_linear: too many rows in one call");
    hipLaunchKernelGGL(dense_f32_kernel, dim3((unsigned)cdiv(d->N, 64), (unsigned)cdiv(d->M, 64)), dim3(256), 0, st,
                       (const float*)d->x, d->ldx, (const float*)d->w, (float*)d->y, d->ldy, d->M, d->K, d->N);
    TNX_CHECK_LAUNCH("dense_f32");
    return TNX_OK;
  }
  TNX_REQUIRE(d->K % kDenseKT == 0, "dense_linear: K=%lld must be a multiple of 128 (zero-pad)", (long long)d->K);
  TNX_REQUIRE(d->epilogue == TNX_EPI_STORE || d->epilogue == TNX_EPI_F32 || d->epilogue == TNX_EPI_GELU_MUL,
              "dense_linear: bad epilogue %d", d->epilogue);
  TNX_REQUIRE(d->epilogue == TNX_EPI_F32 || d->split_k > 1 || d->N % 16 == 0, "dense_linear: N=%lld must be a multiple of 16", (long long)d->N);
  if (d->epilogue == TNX_EPI_GELU_MUL)
    TNX_REQUIRE(d->N % 32 == 0 && d->split_k <= 1, "dense_linear: GELU_MUL needs N %% 32 == 0 and no k split");
  const int64_t ncols = d->epilogue == TNX_EPI_GELU_MUL ? d->N / 2 : d->N;
  TNX_REQUIRE(d->ldy >= ncols && (d->epilogue == TNX_EPI_F32 || d->split_k > 1 || d->ldy % 8 == 0) && (!d->y_frag || d->ldy % 16 == 0),
              "dense_linear: bad output row stride %lld", (long long)d->ldy);
  TNX_REQUIRE(!(d->y_frag && (d->epilogue == TNX_EPI_F32 || d->split_k > 1)), "dense_linear: fragment-order output is bf16");
  TNX_REQUIRE(d->x_frag || (d->ldx >= d->K && d->ldx % 8 == 0), "dense_linear: bad input row stride %lld", (long long)d->ldx);
  const int split = d->split_k < 1 ? 1 : d->split_k;
  TNX_REQUIRE(split == 1 || d->ws, "dense_linear: split_k > 1 needs a workspace");
  TNX_REQUIRE(((uintptr_t)d->x & 15) == 0 && ((uintptr_t)d->w & 15) == 0, "dense_linear: x and w must be 16-byte aligned");
  // many rows: the 128 x 256 kernel (row-major operands, 32-bit offsets)
  if (!d->x_frag && !d->y_frag && split == 1 && d->M > 64 && d->ldx == d->K && d->N % 16 == 0 &&
      cdiv(d->N, 256) * (d->K / kDenseKT) * 65536 < (int64_t)1 << 31)
    return tnx_internal_wide_dense(st, d->M, d->K, d->N, (const uint16_t*)d->x, (const uint16_t*)d->w, d->epilogue, d->y,
                                   d->ldy);
  DenseArgs a;
  a.M = d->M; a.K = d->K; a.N = d->N; a.ldy = d->ldy; a.ldx = d->ldx;
  a.x = (const uint16_t*)d->x; a.w = (const uint16_t*)d->w; a.y = d->y; a.ws = d->ws;
  a.epilogue = d->epilogue; a.x_frag = d->x_frag; a.y_frag = d->y_frag; a.split_k = split;
  const int rt = d->M <= 32 ? 1 : d->M <= 64 ? 2 : 4;
  TNX_REQUIRE(cdiv(d->M, 32 * rt) <= 65535 && split <= 65535, "dense_linear: too many rows or splits in one call");
  const dim3 grid((unsigned)cdiv(d->N, 64), (unsigned)cdiv(d->M, 32 * rt), (unsigned)split);
  if (rt == 1) hipLaunchKernelGGL(dense_rows_kernel<1>, grid, dim3(256), 0, st, a);
  else if (rt == 2) hipLaunchKernelGGL(dense_rows_kernel<2>, grid, dim3(256), 0, st, a);
  else hipLaunchKernelGGL(dense_rows_kernel<4>, grid, dim3(256), 0, st, a);
  TNX_CHECK_LAUNCH("dense_rows");
  return TNX_OK;
}
