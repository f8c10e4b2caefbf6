// Mixture of experts: routing, the plan that sorts (token, choice) entries by expert, the expert linears over that plan,
// and the weighted sum.  Compiled for every element type (the fp32 build has its linears in linear_f32.hip).
#include "moe.h"

namespace {

constexpr int RT_WAVES = 4;
constexpr int RT_MAX_E = 1024;

// One wave per token: z = scale * logit + bias, the `top` largest (the lower index on ties), softmax over those.
__global__ __launch_bounds__(RT_WAVES* WAVE) void moe_route_kernel(int32_t* __restrict__ pick, float* __restrict__ weight,
                                                                  const float* __restrict__ logits, int ld, const float* __restrict__ bias,
                                                                  float scale, int T, int E, int top) {
  __shared__ float zs[RT_WAVES][RT_MAX_E];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int t = blockIdx.x * RT_WAVES + wave;
  if (t >= T) return;                       // no barrier below: the waves are independent
  float* z = zs[wave];
  for (int e = lane; e < E; e += WAVE) z[e] = fmaf(logits[(size_t)t * ld + e], scale, bias[e]);
  float z0 = 0.f, sum = 0.f;
  for (int k = 0; k < top; ++k) {
    float bv = -INFINITY;
    int bi = 0x7fffffff;
    for (int e = lane; e < E; e += WAVE) {  // a lane reads and marks only its own entries
      const float v = z[e];
      if (v > bv) {
        bv = v;
        bi = e;
      }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(bv, o, WAVE);
      const int oi = __shfl_xor(bi, o, WAVE);
      if (ov > bv || (ov == bv && oi < bi)) {
        bv = ov;
        bi = oi;
      }
    }
    if (bi >= E) bi = k;                    // only if the logits are not numbers
    if (k == 0) z0 = bv;
    const float ex = expf(bv - z0);
    sum += ex;
    if (lane == (bi & 63)) z[bi] = -INFINITY;
    if (lane == 0) {
      pick[(size_t)t * top + k] = bi;
      weight[(size_t)t * top + k] = ex;
    }
  }
  // lane 0 wrote the exponentials and scales them itself
  if (lane == 0)
    for (int k = 0; k < top; ++k) weight[(size_t)t * top + k] /= sum;
}

constexpr int PL_THREADS = 1024;
constexpr int PL_MAX_E = RT_MAX_E;

// The experts of a pass's entries: chosen by a router, or looked up by token id.
struct PlanSource {
  const int32_t* pick;      // [n] ...
  const int32_t* table;     // ... or, if given, [layers, V, top]
  const int32_t* ids;       // [n / top]
  int V, top, E;
  __device__ __forceinline__ int operator()(int i) const {
    if (!table) return pick[i];
    const int t = i / top, id = ids[t];
    const int e = table[((size_t)blockIdx.x * V + (id >= 0 && id < V ? id : 0)) * top + i - t * top];
    return e >= 0 && e < E ? e : 0;
  }
};

// Counting sort of the entries by expert, one workgroup (per layer, with tables).  The order of an expert's entries among
// themselves may differ from run to run; nothing depends on it (every row of a tile is computed by itself).
__global__ __launch_bounds__(PL_THREADS) void moe_plan_kernel(int32_t* __restrict__ perm, int4* __restrict__ tiles, int32_t* __restrict__ n_tiles,
                                                              PlanSource pick, int n, int E, int tile_rows, int perm_stride, int tiles_stride) {
  __shared__ int count[PL_MAX_E], first[PL_MAX_E], tile0[PL_MAX_E];
  perm += (size_t)blockIdx.x * perm_stride;
  tiles += (size_t)blockIdx.x * tiles_stride;
  n_tiles += 2 * blockIdx.x;
  for (int e = threadIdx.x; e < E; e += PL_THREADS) count[e] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < n; i += PL_THREADS) atomicAdd(&count[pick(i)], 1);
  __syncthreads();
  if (threadIdx.x < WAVE) {                 // one wave scans, 64 experts at a time
    const int lane = threadIdx.x;
    int base = 0, tbase = 0;
    for (int e0 = 0; e0 < E; e0 += WAVE) {
      const int c = e0 + lane < E ? count[e0 + lane] : 0, cp = (c + 15) & ~15;
      const int nt = (c + tile_rows - 1) / tile_rows;
      int s = cp, ts = nt;
#pragma unroll
      for (int o = 1; o < WAVE; o <<= 1) {
        const int a = __shfl_up(s, o, WAVE), b = __shfl_up(ts, o, WAVE);
        if (lane >= o) {
          s += a;
          ts += b;
        }
      }
      if (e0 + lane < E) {
        first[e0 + lane] = base + s - cp;
        tile0[e0 + lane] = tbase + ts - nt;
      }
      base += __shfl(s, WAVE - 1, WAVE);
      tbase += __shfl(ts, WAVE - 1, WAVE);
    }
    if (lane == 0) {
      n_tiles[0] = tbase;
      n_tiles[1] = base;
    }
  }
  __syncthreads();
  for (int e = threadIdx.x; e < E; e += PL_THREADS) {
    const int c = count[e];
    for (int i = 0, k = 0; i < c; i += tile_rows, ++k) tiles[tile0[e] + k] = make_int4(e, first[e] + i, c - i < tile_rows ? c - i : tile_rows, 0);
    for (int i = c; i & 15; ++i) perm[first[e] + i] = -1;
    count[e] = 0;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < n; i += PL_THREADS) {
    const int e = pick(i);
    perm[first[e] + atomicAdd(&count[e], 1)] = i;
  }
}

// x[t, :] += parts, then sum_k weight[t, k] * y[t * top + k, :], choices in order; out_frag: the result once more, rounded to
// the element type, in fragment order
__global__ __launch_bounds__(256) void moe_combine_kernel(float* __restrict__ x, const float* __restrict__ part, int n_part, size_t part_stride,
                                                          const elt* __restrict__ y, const float* __restrict__ weight, int top, int N,
                                                          elt* __restrict__ out_frag, int frag_tt) {
  const int t = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 4;
  if (c >= N) return;
  f32x4* p = reinterpret_cast<f32x4*>(x + (size_t)t * N + c);
  f32x4 xv = *p;
  for (int q = 0; q < n_part; ++q) xv += *reinterpret_cast<const f32x4*>(part + q * part_stride + (size_t)t * N + c);
  f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k = 0; k < top; ++k) {
    const float w = weight[(size_t)t * top + k];
    const eltx4 v = *reinterpret_cast<const eltx4*>(y + ((size_t)t * top + k) * N + c);
#pragma unroll
    for (int e = 0; e < 4; ++e) s[e] = fmaf(w, (float)v[e], s[e]);
  }
  xv += s;
  *p = xv;
  if (out_frag) *reinterpret_cast<eltx4*>(out_frag + frag_offset(t, c, frag_tt)) = eltx4{(elt)xv[0], (elt)xv[1], (elt)xv[2], (elt)xv[3]};
}

#ifndef MLORA_ELT_F32
struct MoeLinear {
  elt* y;
  const elt* x;
  const elt* W;             // packed, one [N, K] block per expert
  size_t w_elems;
  int K, N, top, up, act;
  float alpha;
};

__device__ __forceinline__ eltx4 moe_out(f32x4 s, const MoeLinear& a) {
  eltx4 o;
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    float v = s[q] * a.alpha;
    if (a.act == MLORA_ACT_RELU2) {
      v = fmaxf(v, 0.f);
      v = v * v;
    }
    o[q] = (elt)v;
  }
  return o;
}

// Tiles of 16 entries (a decode step: a few tokens per expert): the weights are what is read.  A workgroup takes 16 NT rows
// of one expert, its waves split K, the partial tiles meet in LDS in wave order.
constexpr int MG_WAVES = 8;
// GLU: the weights are gate rows, then up rows (a.N of each); a workgroup takes NT / 2 tiles of both and stores their product.
template <int NT, int PIPE, bool GLU = false>
__global__ __launch_bounds__(MG_WAVES* WAVE, 2) void moe_gemv_kernel(MoeLinear a, MoePlan plan) {
  if ((int)blockIdx.y >= *plan.n_tiles) return;
  __shared__ f32x4 red[MG_WAVES][NT][WAVE];
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int4 tile = plan.tiles[blockIdx.y];
  constexpr int NO = GLU ? NT / 2 : NT;       // row tiles of the output
  const int KB = a.K / 32, ntiles = a.N / 16, nt0 = blockIdx.x * NO;
  const int i16 = lane & 15;
  const int place = tile.y + (i16 < tile.z ? i16 : tile.z - 1);
  const int entry = plan.perm[place];
  const elt* xp = a.x + (size_t)(a.up ? entry / a.top : place) * a.K + (lane >> 4) * 8;
  const elt* wp = a.W + tile.x * a.w_elems + lane * 8;
  int woff[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int nt = nt0 + (GLU ? i >> 1 : i);
    woff[i] = ((nt < ntiles ? nt : ntiles - 1) + (GLU && (i & 1) ? ntiles : 0)) * KB * 512;
  }
  f32x4 acc[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int S = (KB - wave + MG_WAVES - 1) / MG_WAVES;
  eltx8 w[PIPE][NT], b[PIPE];
  auto load = [&](int u, int s) {
    const int ks = s < S ? wave + MG_WAVES * s : 0;
#pragma unroll
    for (int i = 0; i < NT; ++i) w[u][i] = ld8(wp + woff[i] + ks * 512);
    b[u] = ld8(xp + ks * 32);
    if (s >= S) b[u] = eltx8{0, 0, 0, 0, 0, 0, 0, 0};     // past this wave's share: valid addresses, no contribution
  };
#pragma unroll
  for (int u = 0; u < PIPE; ++u) load(u, u);
  for (int s0 = 0; s0 < S; s0 += PIPE)
#pragma unroll
    for (int u = 0; u < PIPE; ++u) {
#pragma unroll
      for (int i = 0; i < NT; ++i) acc[i] = mfma_16x16x32(w[u][i], b[u], acc[i]);
      load(u, s0 + u + PIPE);
    }
#pragma unroll
  for (int i = 0; i < NT; ++i) red[wave][i][lane] = acc[i];
  __syncthreads();
  for (int e = threadIdx.x; e < NO * WAVE; e += MG_WAVES * WAVE) {
    const int i = e >> 6, sl = e & 63, row = sl & 15;
    const int n = (nt0 + i) * 16 + (sl >> 4) * 4;
    if (row >= tile.z || n >= a.N) continue;
    const int p = tile.y + row;
    if constexpr (GLU) {
      f32x4 sg = red[0][2 * i][sl], su = red[0][2 * i + 1][sl];
#pragma unroll
      for (int q = 1; q < MG_WAVES; ++q) {
        sg += red[q][2 * i][sl];
        su += red[q][2 * i + 1][sl];
      }
      eltx4 o;
#pragma unroll
      for (int q = 0; q < 4; ++q) o[q] = (elt)glu<MLORA_GLU_SILU>(sg[q], su[q], GluArgs());
      *reinterpret_cast<eltx4*>(a.y + (size_t)p * a.N + n) = o;
      continue;
    }
    f32x4 s = red[0][i][sl];
#pragma unroll
    for (int q = 1; q < MG_WAVES; ++q) s += red[q][i][sl];
    *reinterpret_cast<eltx4*>(a.y + (size_t)(a.up ? p : plan.perm[p]) * a.N + n) = moe_out(s, a);
  }
}

// the token rows of the places, in fragment order: a wave copies one fragment (16 places x 32 columns)
constexpr int MM_ROWS = 256;
__global__ __launch_bounds__(256) void moe_gather_kernel(elt* __restrict__ xf, const elt* __restrict__ x, const int32_t* __restrict__ perm,
                                                         const int32_t* __restrict__ n_tiles, int x_tt, int K, int top) {
  const int lane = threadIdx.x & 63, ks = blockIdx.x * 4 + (threadIdx.x >> 6), tt = blockIdx.y;
  if (tt * 16 >= n_tiles[1] || ks * 32 >= K) return;
  const int entry = perm[tt * 16 + (lane & 15)];
  eltx8 v = eltx8{0, 0, 0, 0, 0, 0, 0, 0};
  if (entry >= 0) v = ld8(x + (size_t)(entry / top) * K + ks * 32 + (lane >> 4) * 8);
  st8(xf + ((size_t)ks * x_tt + tt) * 512 + lane * 8, v);
}
#endif

}  // namespace

extern "C" int mlora_moe_route(int32_t* pick, float* weight, const float* logits, int ld, const float* bias, float scale, int T, int E, int top,
                               void* stream) {
  MLORA_CHECK(pick && weight && logits && bias, MLORA_ERR_INVALID, "moe_route: null pointer");
  MLORA_CHECK(T >= 0 && E > 0 && E <= RT_MAX_E && top > 0 && top <= E && ld >= E, MLORA_ERR_UNSUPPORTED,
              "moe_route: need 0 < top <= experts <= %d (T=%d E=%d top=%d)", RT_MAX_E, T, E, top);
  if (T == 0) return MLORA_OK;
  hipLaunchKernelGGL(moe_route_kernel, dim3(ceil_div(T, RT_WAVES)), dim3(RT_WAVES * WAVE), 0, (hipStream_t)stream, pick, weight, logits, ld, bias,
                     scale, T, E, top);
  return mlora_launch_status("moe_route");
}

// places per expert tile for this many entries (the fp32 build has one size)
extern "C" int mlora_moe_tile_rows(int T, int E, int top) {
#ifdef MLORA_ELT_F32
  return 64;
#else
  return E > 0 && (long)T * top > 16L * E ? MM_ROWS : 16;
#endif
}

// upper bounds, whatever the routing: tiles, and places (a multiple of 16)
extern "C" int mlora_moe_max_tiles(int T, int E, int top) {
  if (T <= 0 || E <= 0 || top <= 0) return 0;
  const long n = (long)T * top;
  return (int)(n / mlora_moe_tile_rows(T, E, top) + (n < E ? n : E));
}

extern "C" int mlora_moe_max_places(int T, int E, int top) {
  if (T <= 0 || E <= 0 || top <= 0) return 0;
  const long n = (long)T * top;
  return (int)((n + 15 * (n < E ? n : E) + 15) / 16 * 16);
}

extern "C" int mlora_moe_plan(int32_t* perm, int32_t* tiles, int32_t* n_tiles, const int32_t* pick, int T, int E, int top, void* stream) {
  MLORA_CHECK(perm && tiles && n_tiles && pick && ((uintptr_t)tiles & 15) == 0, MLORA_ERR_INVALID, "moe_plan: null or unaligned pointer");
  MLORA_CHECK(T > 0 && E > 0 && E <= PL_MAX_E && top > 0 && (long)T * top < 0x7fffffffL, MLORA_ERR_UNSUPPORTED,
              "moe_plan: need experts <= %d (T=%d E=%d top=%d)", PL_MAX_E, T, E, top);
  const PlanSource src = {pick, nullptr, nullptr, 0, top, E};
  hipLaunchKernelGGL(moe_plan_kernel, dim3(1), dim3(PL_THREADS), 0, (hipStream_t)stream, perm, (int4*)tiles, n_tiles, src, T * top, E,
                     mlora_moe_tile_rows(T, E, top), 0, 0);
  return mlora_launch_status("moe_plan");
}

extern "C" int mlora_moe_table_plan(int32_t* perm, int32_t* tiles, int32_t* n_tiles, const int32_t* table, const int32_t* ids, int layers, int V, int T,
                                    int E, int top, void* stream) {
  MLORA_CHECK(perm && tiles && n_tiles && table && ids && ((uintptr_t)tiles & 15) == 0, MLORA_ERR_INVALID, "moe_table_plan: null or unaligned pointer");
  MLORA_CHECK(layers > 0 && V > 0 && T > 0 && E > 0 && E <= PL_MAX_E && top > 0 && (long)T * top < 0x7fffffffL, MLORA_ERR_UNSUPPORTED,
              "moe_table_plan: need experts <= %d (layers=%d V=%d T=%d E=%d top=%d)", PL_MAX_E, layers, V, T, E, top);
  const PlanSource src = {nullptr, table, ids, V, top, E};
  hipLaunchKernelGGL(moe_plan_kernel, dim3(layers), dim3(PL_THREADS), 0, (hipStream_t)stream, perm, (int4*)tiles, n_tiles, src, T * top, E,
                     mlora_moe_tile_rows(T, E, top), mlora_moe_max_places(T, E, top), mlora_moe_max_tiles(T, E, top));
  return mlora_launch_status("moe_table_plan");
}

extern "C" int mlora_moe_combine(float* x, const float* part, int n_part, const void* y, const float* weight, int T, int top, int N,
                                 void* out_frag, void* stream) {
  MLORA_CHECK(x && y && weight && n_part >= 0 && (n_part == 0 || part), MLORA_ERR_INVALID, "moe_combine: null pointer");
  MLORA_CHECK(T >= 0 && T <= 65535 && top > 0 && N > 0 && N % 4 == 0 && (!out_frag || (N % 32 == 0 && sizeof(elt) == 2)), MLORA_ERR_UNSUPPORTED,
              "moe_combine: T=%d top=%d N=%d", T, top, N);
  if (T == 0) return MLORA_OK;
  hipLaunchKernelGGL(moe_combine_kernel, dim3(ceil_div(N, 1024), T), dim3(256), 0, (hipStream_t)stream, x, part, n_part, (size_t)T * N,
                     (const elt*)y, weight, top, N, (elt*)out_frag, mlora_frag_tiles(T));
  return mlora_launch_status("moe_combine");
}

#ifndef MLORA_ELT_F32
extern "C" int mlora_moe_linear(void* y, const void* x, const void* W, const int32_t* perm, const int32_t* tiles, const int32_t* n_tiles,
                                int tile_rows, int max_tiles, int places, int T, int K, int N, int top, int stage, int act, float alpha,
                                void* workspace, size_t workspace_elems, void* stream) {
  MLORA_CHECK(y && x && W && perm && tiles && n_tiles, MLORA_ERR_INVALID, "moe_linear: null pointer");
  MLORA_CHECK(T >= 0 && K > 0 && K % 32 == 0 && N > 0 && N % 16 == 0 && top > 0 && max_tiles >= 0 && max_tiles <= 65535 &&
                  (long)N * K < (1L << (act == MLORA_ACT_GLU ? 30 : 31)) && (tile_rows == 16 || tile_rows == MM_ROWS) && places % 16 == 0 && places / 16 <= 65535,
              MLORA_ERR_UNSUPPORTED, "moe_linear: need K %% 32 == 0, N %% 16 == 0 (T=%d K=%d N=%d tiles=%d)", T, K, N, max_tiles);
  MLORA_CHECK(act != MLORA_ACT_GLU || (stage == MLORA_MOE_UP && alpha == 1.f), MLORA_ERR_UNSUPPORTED, "moe_linear: a gated product is the up stage's, unscaled");
  if (T == 0 || max_tiles == 0) return MLORA_OK;
  MoePlan p;
  p.perm = perm; p.tiles = (const int4*)tiles; p.n_tiles = n_tiles;
  hipStream_t s = (hipStream_t)stream;
  if (tile_rows == MM_ROWS) {
    MLORA_CHECK(K % 64 == 0 && N % 32 == 0 && (((uintptr_t)x | (uintptr_t)y | (uintptr_t)workspace) & 15) == 0, MLORA_ERR_UNSUPPORTED,
                "moe_linear: 256-place tiles need K %% 64 == 0, N %% 32 == 0, aligned operands (K=%d N=%d)", K, N);
    MLORA_CHECK(stage == MLORA_MOE_UP ? act != MLORA_ACT_NONE : act == MLORA_ACT_NONE, MLORA_ERR_UNSUPPORTED,
                "moe_linear: over 256-place tiles the up stage ends with its activation, the down stage has none");
    const void* xf = x;
    if (stage == MLORA_MOE_UP) {
      MLORA_CHECK(workspace && workspace_elems >= (size_t)places * K, MLORA_ERR_WORKSPACE, "moe_linear: workspace of %zu elements needed", (size_t)places * K);
      hipLaunchKernelGGL(moe_gather_kernel, dim3(ceil_div(K, 128), places / 16), dim3(256), 0, s, (elt*)workspace, (const elt*)x, perm, n_tiles,
                         places / 16, K, top);
      xf = workspace;
    }
    return mlora_gemm_grouped(y, xf, places / 16, W, p, max_tiles, K, N, act, alpha, stream);
  }
  MoeLinear a;
  a.y = (elt*)y; a.x = (const elt*)x; a.W = (const elt*)W; a.w_elems = (size_t)N * K * (act == MLORA_ACT_GLU ? 2 : 1);
  a.K = K; a.N = N; a.top = top; a.up = stage == MLORA_MOE_UP; a.act = act; a.alpha = alpha;
  if (act == MLORA_ACT_GLU) hipLaunchKernelGGL((moe_gemv_kernel<2, 4, true>), dim3(N / 16, max_tiles), dim3(MG_WAVES * WAVE), 0, s, a, p);
  else hipLaunchKernelGGL((moe_gemv_kernel<2, 4>), dim3(ceil_div(N, 32), max_tiles), dim3(MG_WAVES * WAVE), 0, s, a, p);
  return mlora_launch_status("moe_linear");
}
#endif
