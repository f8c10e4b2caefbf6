// Linear layers of the fp32 build:  y[T, N] (=|+=) alpha x[T, K] . W[N, K]^T  in IEEE fp32 on the vector ALUs, plain, per
// head (a batch of small matrices) or per expert (token tiles of a routing plan).  64 x 64 output blocks, operands staged
// through LDS, sums in ascending k.
#include "common.h"
#include "moe.h"

namespace {

constexpr int FB = 64;       // block side
constexpr int FK = 16;       // k per stage

struct F32Linear {
  float* y;
  const float* x;
  const float* W;
  long ldx, ldy;
  long hx, hy;               // head strides of x and y (blockIdx.z = head; the weights of a head are [N, K] blocks)
  int T, K, N;
  float alpha;
  int accumulate, act;       // act: MLORA_ACT_*
  int gather, scatter, top;  // expert tiles (blockIdx.y = tile): gather: x row = entry / top; scatter: y row = entry
};

__global__ __launch_bounds__(256) void linear_f32_kernel(F32Linear a, MoePlan plan, int grouped) {
  __shared__ float xs[FK][FB + 4], ws[FK][FB + 4];
  const int n0 = blockIdx.x * FB;
  int t0 = blockIdx.y * FB, t1 = a.T;
  const float* W = a.W + (size_t)blockIdx.z * a.N * a.K;
  const float* x = a.x + blockIdx.z * a.hx;
  float* y = a.y + blockIdx.z * a.hy;
  if (grouped) {
    if ((int)blockIdx.y >= *plan.n_tiles) return;
    const int4 tile = plan.tiles[blockIdx.y];
    W = a.W + (size_t)tile.x * a.N * a.K;
    t0 = tile.y;
    t1 = tile.y + tile.z;
  }
  const int tx = threadIdx.x & 15, ty = threadIdx.x >> 4;
  float acc[4][4] = {};
  // loader: thread -> row threadIdx / 4, four k at (threadIdx % 4) * 4
  const int lr = threadIdx.x >> 2, lk = (threadIdx.x & 3) * 4;
  int xrow = t0 + lr < t1 ? t0 + lr : t1 - 1;
  if (grouped && a.gather) xrow = plan.perm[xrow] / a.top;
  const int wrow = n0 + lr < a.N ? n0 + lr : a.N - 1;
  for (int k0 = 0; k0 < a.K; k0 += FK) {
    const f32x4 xv = *reinterpret_cast<const f32x4*>(x + xrow * a.ldx + k0 + lk);
    const f32x4 wv = *reinterpret_cast<const f32x4*>(W + (size_t)wrow * a.K + k0 + lk);
    __syncthreads();
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      xs[lk + e][lr] = xv[e];
      ws[lk + e][lr] = wv[e];
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < FK; ++k) {
      const f32x4 xf = *reinterpret_cast<const f32x4*>(&xs[k][ty * 4]), wf = *reinterpret_cast<const f32x4*>(&ws[k][tx * 4]);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(xf[i], wf[j], acc[i][j]);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    int t = t0 + ty * 4 + i;
    if (t >= t1) continue;
    if (grouped && a.scatter) t = plan.perm[t];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int n = n0 + tx * 4 + j;
      if (n >= a.N) continue;
      float v = acc[i][j] * a.alpha;
      if (a.act == MLORA_ACT_RELU2) {
        v = fmaxf(v, 0.f);
        v = v * v;
      }
      float* p = y + t * a.ldy + n;
      *p = a.accumulate ? *p + v : v;
    }
  }
}

int launch(const char* who, const F32Linear& a, const MoePlan& plan, int grouped, int row_blocks, int heads, void* stream) {
  MLORA_CHECK(a.K % FK == 0 && a.ldx % 4 == 0 && a.hx % 4 == 0 && row_blocks <= 65535 && heads <= 65535, MLORA_ERR_UNSUPPORTED,
              "%s: need K %% 16 == 0 and rows aligned to 16 bytes (T=%d K=%d N=%d)", who, a.T, a.K, a.N);
  hipLaunchKernelGGL(linear_f32_kernel, dim3(ceil_div(a.N, FB), row_blocks, heads), dim3(256), 0, (hipStream_t)stream, a, plan, grouped);
  return mlora_launch_status(who);
}

}  // namespace

extern "C" int mlora_linear(void* y, int y_dtype, int mode, const void* x, int ldx, const void* W, int T, int K, int N, void* stream) {
  MLORA_CHECK(y && x && W && T >= 0 && K > 0 && N > 0 && ldx >= K, MLORA_ERR_INVALID, "linear: null pointer or bad shape T=%d K=%d N=%d", T, K, N);
  if (T == 0) return MLORA_OK;
  F32Linear a = {};
  a.y = (float*)y; a.x = (const float*)x; a.W = (const float*)W;
  a.ldx = ldx; a.ldy = N; a.T = T; a.K = K; a.N = N; a.alpha = 1.f; a.accumulate = mode == MLORA_ACCUMULATE;
  return launch("linear", a, MoePlan(), 0, ceil_div(T, FB), 1, stream);
}

extern "C" int mlora_head_linear(void* y, int y_layout, long ldy, long head_y, const void* x, long ldx, long head_x, const void* W, int heads, int T,
                                 int K, int N, float alpha, void* stream) {
  MLORA_CHECK(y && x && W && T >= 0 && K > 0 && N > 0 && heads > 0, MLORA_ERR_INVALID, "head_linear: null pointer or bad shape");
  MLORA_CHECK(y_layout == MLORA_ROWMAJOR, MLORA_ERR_UNSUPPORTED, "head_linear: fragment order is for 16-bit elements");
  if (T == 0) return MLORA_OK;
  F32Linear a = {};
  a.y = (float*)y; a.x = (const float*)x; a.W = (const float*)W;
  a.ldx = ldx; a.ldy = ldy; a.hx = head_x; a.hy = head_y; a.T = T; a.K = K; a.N = N; a.alpha = alpha;
  return launch("head_linear", a, MoePlan(), 0, ceil_div(T, FB), heads, stream);
}

extern "C" int mlora_moe_linear(void* y, const void* x, const void* W, const int32_t* perm, const int32_t* tiles, const int32_t* n_tiles,
                                int tile_rows, int max_tiles, int places, int T, int K, int N, int top, int stage, int act, float alpha,
                                void* workspace, size_t workspace_elems, void* stream) {
  MLORA_CHECK(y && x && W && perm && tiles && n_tiles && T >= 0 && K > 0 && N > 0 && top > 0 && tile_rows == FB, MLORA_ERR_INVALID,
              "moe_linear: null pointer or bad shape (tile_rows=%d)", tile_rows);
  (void)places; (void)workspace; (void)workspace_elems;      // the matrix-core form's
  if (T == 0) return MLORA_OK;
  F32Linear a = {};
  a.y = (float*)y; a.x = (const float*)x; a.W = (const float*)W;
  a.ldx = K; a.ldy = N; a.T = T * top; a.K = K; a.N = N; a.alpha = alpha; a.act = act; a.top = top;
  a.gather = stage == MLORA_MOE_UP;
  a.scatter = stage == MLORA_MOE_DOWN;
  MoePlan p;
  p.perm = perm; p.tiles = (const int4*)tiles; p.n_tiles = n_tiles;
  return launch("moe_linear", a, p, 1, max_tiles, 1, stream);
}
