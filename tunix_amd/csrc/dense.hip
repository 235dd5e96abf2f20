// Linears with dense weights (bf16 or fp32) for decoders whose weights are not quantised.
//
// bf16: the weights live in HBM once, in the fragment order of tnx_dense_expand.  Calls with many
// rows take the 128 x 256 kernel of qgemm_wide.h; calls with few rows take dense_rows_kernel below,
// which streams the same copy.  fp32: a plain tiled kernel in true 32-bit arithmetic.
//
// Two forms run several weights of one shape in a launch: a batch (every row through every weight, e.g.
// one per head) and experts (a row goes to the weights its routes name, rows sorted by expert).
#include <string.h>

#include <mutex>
#include <type_traits>

#include "decoder.h"

int tnx_internal_wide_dense(hipStream_t st, int64_t M, int64_t K, int64_t N, const uint16_t* x, const uint16_t* w,
                            int epilogue, void* y, int64_t ldy);
int tnx_internal_wide_dense_grouped(hipStream_t st, int64_t n_routes, int64_t K, int64_t N, const uint16_t* x, const uint16_t* w,
                                    int epilogue, void* y, int64_t ldy, int n_experts, const int32_t* offsets,
                                    const int32_t* sorted_route, int x_div);

namespace {

struct DenseArgs {
  int64_t M, K, N, ldy, ldx;
  const uint16_t* x;
  const uint16_t* w;
  void* y;
  float* ws;
  int epilogue, x_frag, y_frag, split_k;
  int64_t x_stride, w_stride, y_stride;   // batch, experts: elements from one weight's operands to the next
  int n_experts, x_div;
  const int32_t* offsets;
  const int32_t* sorted_route;
  int row_xcd;             // grid x counts eight row blocks times the column blocks: a row block's stay on one XCD, whose L2 holds its rows
};
constexpr int kPlain = 0, kBatch = 1, kExperts = 2;

// Block `blk` of `rows` rows of the expert-sorted routes -> its expert, first row and end; false past the
// last block.  Same result in every wave.
__device__ __forceinline__ bool find_block(const int32_t* offsets, int n_experts, int rows, int blk, int& expert, int& first_row, int& end_row) {
  const int lane = threadIdx.x & 63;
  int carry = 0, found_e = -1, found_rb = 0;
  for (int base = 0; base < n_experts; base += 64) {
    const int e = base + lane;
    int nb = 0;
    if (e < n_experts) nb = (offsets[e + 1] - offsets[e] + rows - 1) / rows;
    int incl = nb;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int t = __shfl_up(incl, o, 64);
      if (lane >= o) incl += t;
    }
    const int first = carry + incl - nb;
    const uint64_t hit = __ballot(nb > 0 && blk >= first && blk < first + nb);
    if (hit) {
      const int l = __ffsll((long long)hit) - 1;
      found_e = base + l;
      found_rb = blk - __shfl(first, l, 64);
      break;
    }
    carry += __shfl(incl, 63, 64);
  }
  if (found_e < 0) return false;
  expert = __builtin_amdgcn_readfirstlane(found_e);
  first_row = offsets[expert] + __builtin_amdgcn_readfirstlane(found_rb) * rows;
  end_row = offsets[expert + 1];
  return true;
}

__device__ __forceinline__ f32x4 square_relu(f32x4 v) {
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = fmaxf(v[e], 0.f) * fmaxf(v[e], 0.f);
  return v;
}

constexpr int kDenseKT = 128;   // k-tile of the fragment layout: eight 16-deep slabs

// A work-group of four waves owns 32 * RT rows x 64 columns (two 32-column groups); its waves take
// the k-tiles of the work-group's k range in turn and meet through LDS at the end.  A slab of a
// column group is one 16-byte load per lane (1 KB per wave, contiguous), eight slabs ahead of
// their use in a register ring; activations in fragment order come the same way from L2.
// Products are formed transposed (weights as the MFMA's A operand): a lane owns runs of four
// consecutive columns of one row.
// MODE kBatch: blockIdx.z is the weight; kExperts: blockIdx.y is a block of 32 RT routes of one expert.
template <int RT, int MODE>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(RT == 1 ? 3 : 1, RT == 4 ? 1 : RT == 2 ? 2 : 4)))
void dense_rows_kernel(const DenseArgs a) {
  constexpr int CG = 2, XD = RT == 1 ? 8 : 4;   // column groups; slabs of activations in flight
  __shared__ __align__(16) float red[4][CG * 16 * 64];
  const int tid = threadIdx.x, lane = tid & 63, l32 = lane & 31, lh = lane >> 5;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  int c64 = blockIdx.x;
  int64_t m0 = (int64_t)blockIdx.y * (32 * RT), m_end = a.M;
  if (MODE == kPlain && a.row_xcd) {
    c64 = blockIdx.x >> 3;
    m0 = ((int64_t)blockIdx.y * 8 + (blockIdx.x & 7)) * (32 * RT);
    if (m0 >= m_end) return;
  }
  int64_t x_at = 0, w_at = 0, y_at = 0;
  if constexpr (MODE == kBatch) {
    x_at = blockIdx.z * a.x_stride;
    w_at = blockIdx.z * a.w_stride;
    y_at = blockIdx.z * a.y_stride;
  }
  if constexpr (MODE == kExperts) {
    int expert, first_row, end_row;
    if (!find_block(a.offsets, a.n_experts, 32 * RT, (int)blockIdx.y, expert, first_row, end_row)) return;
    m0 = first_row;
    m_end = end_row;
    w_at = expert * a.w_stride;
  }
  const int z = MODE == kBatch ? 0 : blockIdx.z;
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
  const u32x4* wb = reinterpret_cast<const u32x4*>(a.w + w_at) + ((int64_t)(c64 >> 2) * ktiles * 8 + (c64 & 3) * 2) * 512 + lane;
  // lane: row l32 of every 32, eight k from 8 lh on; rows past the end repeat the last one
  const int64_t kslabs = a.K / 16;
  const unsigned char* xb = reinterpret_cast<const unsigned char*>(a.x + x_at);
  uint32_t xo[RT];                        // byte offsets (the host checks that they fit)
  int orow[RT];                       // the row this lane stores, -1: none
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) {
    const int r = (int)m0 + rt * 32 + l32, rc = min(r, (int)m_end - 1);
    int row = rc;
    orow[rt] = r < m_end ? r : -1;
    if constexpr (MODE == kExperts) {
      const int route = a.sorted_route[rc];
      row = route / a.x_div;
      if (orow[rt] >= 0) orow[rt] = route;
    }
    xo[rt] = a.x_frag ? ((uint32_t)(row >> 5) * (uint32_t)kslabs << 10) + (lh << 9) + ((row & 31) << 4)
                      : ((uint32_t)row * (uint32_t)a.ldx + lh * 8) * 2;
  }
  const int xstep = a.x_frag ? 1024 : 32;
  auto load_x = [&](int slab, int rt) -> u32x4 { return *reinterpret_cast<const u32x4*>(xb + slab * xstep + xo[rt]); };
  u32x4 wr[8][CG];
  auto load_w = [&](int kt, int u) {
#pragma unroll
    for (int cg = 0; cg < CG; ++cg) wr[u][cg] = wb[((int64_t)kt * 8 + cg) * 512 + u * 64];
  };
  int kt = kt0 + wave;
  if (kt < kt1) {
    u32x4 xr[XD][RT];
    // in the loop's order, so that its counted waits are the same on the way in
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      if (u + XD - 1 >= 8)
#pragma unroll
        for (int rt = 0; rt < RT; ++rt) xr[(u + XD - 1) % XD][rt] = load_x(kt * 8 + u + XD - 9, rt);
      load_w(kt, u);
      __builtin_amdgcn_sched_barrier(0);
    }
    // a tile's products; `more`: the wave has another tile, whose operands are requested meanwhile
    auto tile = [&](auto more) {
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const int n = u + XD - 1;
        if (n < 8 || more)
#pragma unroll
          for (int rt = 0; rt < RT; ++rt) xr[n % XD][rt] = load_x(n < 8 ? kt * 8 + n : kt * 8 + 24 + n, rt);
#pragma unroll
        for (int cg = 0; cg < CG; ++cg)
#pragma unroll
          for (int rt = 0; rt < RT; ++rt) acc[rt][cg] = mfma32(wr[u][cg], xr[u % XD][rt], acc[rt][cg]);
        if (more) load_w(kt + 4, u);
        __builtin_amdgcn_sched_barrier(0);   // (a load sunk to its use would leave nothing in flight)
      }
    };
    for (; kt + 4 < kt1; kt += 4) tile(std::true_type{});
    tile(std::false_type{});
  }

  // the four waves' parts meet, one row tile at a time; wave w then owns one quarter of the tile
  const bool silu = a.epilogue == TNX_EPI_SILU_MUL, mul = a.epilogue == TNX_EPI_GELU_MUL || silu;
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
    const int64_t row = orow[rt];
    if (row < 0) continue;
    if (mul) {
      // a 32-column group is [16 gate | 16 up]: quarters b and b + 2 pair up
      const int cg = wave >> 1, b = wave & 1;
      const f32x4 g = total(cg, b), u = total(cg, b + 2);
      const int64_t col = (int64_t)(c64 * 2 + cg) * 16 + 8 * b + 4 * lh;
      if (col >= a.N / 2) continue;
      float v[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = (silu ? silu_f32(g[e]) : gelu_tanh_f32(g[e])) * u[e];
      const u32x2 pk = {pack2bf(v[0], v[1]), pack2bf(v[2], v[3])};
      uint16_t* y = reinterpret_cast<uint16_t*>(a.y);
      *reinterpret_cast<u32x2*>(y + (a.y_frag ? frag_index(row, col, a.ldy) : row * a.ldy + col)) = pk;
      continue;
    }
#pragma unroll
    for (int cg = 0; cg < CG; ++cg) {
      const f32x4 v = total(cg, wave);
      const int64_t col = (int64_t)(c64 * 2 + cg) * 32 + 8 * wave + 4 * lh;
      if (a.epilogue == TNX_EPI_F32 || a.split_k > 1) {
        float* y = a.split_k > 1 ? a.ws + (int64_t)z * a.M * a.ldy : reinterpret_cast<float*>(a.y) + y_at;
        y += row * a.ldy + col;
        if (col + 4 <= a.N && (a.ldy & 3) == 0) {
          *reinterpret_cast<f32x4*>(y) = v;
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (col + e < a.N) y[e] = v[e];
        }
      } else if (col < a.N) {   // bf16: N is a multiple of 16
        uint16_t* y = reinterpret_cast<uint16_t*>(a.y) + y_at;
        const f32x4 u = a.epilogue == TNX_EPI_RELU2 ? square_relu(v) : v;
        *reinterpret_cast<u32x2*>(y + (a.y_frag ? frag_index(row, col, a.ldy) : row * a.ldy + col)) =
            u32x2{pack2bf(u[0], u[1]), pack2bf(u[2], u[3])};
      }
    }
  }
}

// fp32: 64 x 64 tile, 256 threads, 4 x 4 outputs each; K a multiple of 16
template <int MODE>
__global__ __launch_bounds__(256) void dense_f32_kernel(const DenseArgs a) {
  __shared__ float xs[16][68], wsh[16][68];
  const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
  const int64_t n0 = (int64_t)blockIdx.x * 64, K = a.K, N = a.N, ldy = a.ldy;
  int64_t m0 = (int64_t)blockIdx.y * 64, M = a.M;
  const float* x = reinterpret_cast<const float*>(a.x);
  const float* w = reinterpret_cast<const float*>(a.w);
  float* y = reinterpret_cast<float*>(a.y);
  if constexpr (MODE == kBatch) {
    x += blockIdx.z * a.x_stride;
    w += blockIdx.z * a.w_stride;
    y += blockIdx.z * a.y_stride;
  }
  if constexpr (MODE == kExperts) {
    int expert, first_row, end_row;
    if (!find_block(a.offsets, a.n_experts, 64, (int)blockIdx.y, expert, first_row, end_row)) return;
    m0 = first_row;
    M = end_row;
    w += expert * a.w_stride;
  }
  const int lr = tid >> 2, lk = (tid & 3) * 4;
  int64_t xrow = m0 + lr;
  if constexpr (MODE == kExperts) xrow = xrow < M ? a.sorted_route[xrow] / a.x_div : 0;
  float acc[4][4] = {};
  for (int64_t k0 = 0; k0 < K; k0 += 16) {
    f32x4 xv = f32x4{0.f, 0.f, 0.f, 0.f}, wv = xv;
    if (m0 + lr < M) xv = *reinterpret_cast<const f32x4*>(x + xrow * a.ldx + k0 + lk);
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
  for (int i = 0; i < 4; ++i) {
    int64_t row = m0 + ty * 4 + i;
    if (row >= M) break;
    if constexpr (MODE == kExperts) row = a.sorted_route[row];
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (n0 + tx * 4 + j < N) y[row * ldy + n0 + tx * 4 + j] = a.epilogue == TNX_EPI_RELU2 ? fmaxf(acc[i][j], 0.f) * fmaxf(acc[i][j], 0.f) : acc[i][j];
  }
}

template <int MODE>
void launch_rows(hipStream_t st, const DenseArgs& a, int rt, const dim3& grid) {
  if (rt == 1) hipLaunchKernelGGL((dense_rows_kernel<1, MODE>), grid, dim3(256), 0, st, a);
  else if (rt == 2) hipLaunchKernelGGL((dense_rows_kernel<2, MODE>), grid, dim3(256), 0, st, a);
  else hipLaunchKernelGGL((dense_rows_kernel<4, MODE>), grid, dim3(256), 0, st, a);
}

}  // namespace

extern "C" int tnx_dense_linear(void* stream, const tnx_dense_desc* d) {
  TNX_REQUIRE(d, "dense_linear: null descriptor");
  TNX_REQUIRE(d->M > 0 && d->K > 0 && d->N > 0, "dense_linear: M, K, N must be positive");
  TNX_REQUIRE(d->x && d->w && (d->y || d->split_k > 1), "dense_linear: null pointer");
  TNX_REQUIRE(d->dtype == TNX_BF16 || d->dtype == TNX_F32, "dense_linear: bad dtype %d", d->dtype);
  hipStream_t st = as_stream(stream);
  const bool batch = d->batch > 1, experts = d->n_experts > 0;
  TNX_REQUIRE(!(batch && experts) && ((!batch && !experts) || d->split_k <= 1), "dense_linear: batch, experts and k splits exclude each other");
  TNX_REQUIRE(!batch || (d->batch <= 65535 && !d->x_frag && !d->y_frag), "dense_linear: a batch takes row-major operands");
  TNX_REQUIRE(!experts || (d->offsets && d->sorted_route && d->x_div >= 1 && d->n_experts <= 65535 && !d->y_frag && d->M < ((int64_t)1 << 30)),
              "dense_linear: experts need their offsets and sorted routes");
  DenseArgs a;
  memset(&a, 0, sizeof(a));
  a.M = d->M; a.K = d->K; a.N = d->N; a.ldy = d->ldy; a.ldx = d->ldx;
  a.x = (const uint16_t*)d->x; a.w = (const uint16_t*)d->w; a.y = d->y; a.ws = d->ws;
  a.epilogue = d->epilogue; a.x_frag = d->x_frag; a.y_frag = d->y_frag; a.split_k = d->split_k < 1 ? 1 : d->split_k;
  a.x_stride = d->x_stride; a.w_stride = d->w_stride; a.y_stride = d->y_stride;
  a.n_experts = d->n_experts; a.x_div = d->x_div; a.offsets = d->offsets; a.sorted_route = d->sorted_route;
  if (d->dtype == TNX_F32) {
    TNX_REQUIRE(d->K % 16 == 0 && d->ldx % 4 == 0 && d->ldx >= d->K && d->ldy >= d->N,
                "dense_linear: fp32 needs K %% 16 == 0 and row strides that hold the rows");
    TNX_REQUIRE((d->epilogue == TNX_EPI_STORE || d->epilogue == TNX_EPI_F32 || d->epilogue == TNX_EPI_RELU2) && d->split_k <= 1 && !d->x_frag && !d->y_frag,
                "dense_linear: fp32 stores row-major results only");
    const int64_t blocks = experts ? d->M / 64 + (d->n_experts < d->M ? d->n_experts : d->M) : cdiv(d->M, 64);
    TNX_REQUIRE(blocks <= 65535, "dense_linear: too many rows in one call");
    TNX_REQUIRE(d->x_stride % 4 == 0 && d->w_stride % 4 == 0, "dense_linear: operands of a batch must stay 16-byte aligned");
    const dim3 grid((unsigned)cdiv(d->N, 64), (unsigned)blocks, batch ? (unsigned)d->batch : 1u);
    if (experts) hipLaunchKernelGGL(dense_f32_kernel<kExperts>, grid, dim3(256), 0, st, a);
    else if (batch) hipLaunchKernelGGL(dense_f32_kernel<kBatch>, grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL(dense_f32_kernel<kPlain>, grid, dim3(256), 0, st, a);
    TNX_CHECK_LAUNCH("dense_f32");
    return TNX_OK;
  }
  TNX_REQUIRE(d->K % kDenseKT == 0, "dense_linear: K=%lld must be a multiple of 128 (zero-pad)", (long long)d->K);
  const bool mul = d->epilogue == TNX_EPI_GELU_MUL || d->epilogue == TNX_EPI_SILU_MUL;
  TNX_REQUIRE(d->epilogue == TNX_EPI_STORE || d->epilogue == TNX_EPI_F32 || d->epilogue == TNX_EPI_RELU2 || mul, "dense_linear: bad epilogue %d", d->epilogue);
  TNX_REQUIRE(d->epilogue != TNX_EPI_RELU2 || d->split_k <= 1, "dense_linear: an activation needs whole sums: no k split");
  TNX_REQUIRE(d->epilogue == TNX_EPI_F32 || d->split_k > 1 || d->N % 16 == 0, "dense_linear: N=%lld must be a multiple of 16", (long long)d->N);
  if (mul) TNX_REQUIRE(d->N % 32 == 0 && d->split_k <= 1, "dense_linear: a gated unit needs N %% 32 == 0 and no k split");
  const int64_t ncols = mul ? d->N / 2 : d->N;
  TNX_REQUIRE(d->ldy >= ncols && (d->epilogue == TNX_EPI_F32 || d->split_k > 1 || d->ldy % 8 == 0) && (!d->y_frag || d->ldy % 16 == 0),
              "dense_linear: bad output row stride %lld", (long long)d->ldy);
  TNX_REQUIRE(!(d->y_frag && (d->epilogue == TNX_EPI_F32 || d->split_k > 1)), "dense_linear: fragment-order output is bf16");
  TNX_REQUIRE(d->x_frag || (d->ldx >= d->K && d->ldx % 8 == 0), "dense_linear: bad input row stride %lld", (long long)d->ldx);
  const int split = a.split_k;
  TNX_REQUIRE(split == 1 || d->ws, "dense_linear: split_k > 1 needs a workspace");
  TNX_REQUIRE(((uintptr_t)d->x & 15) == 0 && ((uintptr_t)d->w & 15) == 0, "dense_linear: x and w must be 16-byte aligned");
  TNX_REQUIRE(!batch || (d->x_stride % 8 == 0 && d->w_stride % 8 == 0 && d->y_stride % 4 == 0), "dense_linear: operands of a batch must stay aligned");
  const int64_t x_rows = experts ? cdiv(d->M, (int64_t)d->x_div) : cdiv(d->M, 128) * 128;
  const bool x32 = x_rows * (d->x_frag ? d->K : d->ldx) < (int64_t)1 << 31;
  const bool offsets32 = cdiv(d->N, 256) * (d->K / kDenseKT) * 65536 < (int64_t)1 << 31;
  if (experts) {
    // rows per block: as many as an expert gets on average, and the 128 x 256 kernel from about 24 on (a
    // second block of an expert streams its weights again)
    const int64_t avg = cdiv(d->M, (int64_t)d->n_experts);
    TNX_REQUIRE(d->w_stride == cdiv(d->N, 256) * 256 * d->K, "dense_linear: an expert's weights are one fragment-order copy");
    if (avg > 24 && !d->x_frag && d->ldx == d->K && d->N % 16 == 0 && ncols % 8 == 0 && offsets32 && d->M % d->x_div == 0 &&
        (uint64_t)(d->M / d->x_div) * (uint64_t)d->K * 2 < 0xfffff000ull && ((uintptr_t)d->y & 15) == 0 && d->epilogue != TNX_EPI_F32)
      return tnx_internal_wide_dense_grouped(st, d->M, d->K, d->N, a.x, a.w, d->epilogue, d->y, d->ldy, d->n_experts, d->offsets,
                                             d->sorted_route, d->x_div);
    TNX_REQUIRE(x32, "dense_linear: x must stay below 4 GiB");
    const int rt = avg <= 32 ? 1 : avg <= 64 ? 2 : 4;
    const int64_t blocks = d->M / (32 * rt) + (d->n_experts < d->M ? d->n_experts : d->M);
    TNX_REQUIRE(blocks <= 65535, "dense_linear: too many routes in one call");
    launch_rows<kExperts>(st, a, rt, dim3((unsigned)cdiv(d->N, 64), (unsigned)blocks));
    TNX_CHECK_LAUNCH("dense_rows");
    return TNX_OK;
  }
  // many rows: the 128 x 256 kernel (row-major operands, 32-bit offsets); a few columns would leave its tiles
  // and the device mostly empty: 32 rows per work-group then
  const bool narrow = d->N <= 128 && !mul && d->M > 64 && d->M <= 32 * 65535;
  if (!batch && !narrow && !d->x_frag && !d->y_frag && split == 1 && d->M > 64 && d->ldx == d->K && d->N % 16 == 0 &&
      offsets32)
    return tnx_internal_wide_dense(st, d->M, d->K, d->N, (const uint16_t*)d->x, (const uint16_t*)d->w, d->epilogue, d->y,
                                   d->ldy);
  TNX_REQUIRE(x32, "dense_linear: x must stay below 4 GiB");
  int rt = d->M <= 32 || narrow ? 1 : d->M <= 64 ? 2 : 4;
  while (batch && rt > 1 && cdiv(d->N, 64) * cdiv(d->M, 32 * rt) * d->batch < 512) rt /= 2;
  TNX_REQUIRE(cdiv(d->M, 32 * rt) <= 65535 && split <= 65535, "dense_linear: too many rows or splits in one call");
  dim3 grid((unsigned)cdiv(d->N, 64), (unsigned)cdiv(d->M, 32 * rt), batch ? (unsigned)d->batch : (unsigned)split);
  if (!batch && narrow && grid.x > 1 && grid.y >= 64) {
    a.row_xcd = 1;
    grid = dim3(grid.x * 8, (unsigned)cdiv((int64_t)grid.y, 8), grid.z);
  }
  if (batch) launch_rows<kBatch>(st, a, rt, grid);
  else launch_rows<kPlain>(st, a, rt, grid);
  TNX_CHECK_LAUNCH("dense_rows");
  return TNX_OK;
}
