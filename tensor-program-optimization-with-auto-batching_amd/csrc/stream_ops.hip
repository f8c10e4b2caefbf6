// Row operators of decoders with an fp32 residual stream: the one-number norm and a per-layer token input; the elementwise
// norm ahead of and behind a sublayer, with the mixes of neighbouring tokens.  Compiled for every element type.
#include "common.h"

namespace {

constexpr int SN_THREADS = 256;

__device__ __forceinline__ float sn_block_sum(float v, float* lds) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) lds[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int w = 0; w < SN_THREADS / WAVE; ++w) s += lds[w];
  return s;
}

struct StreamNorm {
  float* x;               // [T, Hp] residual stream, columns H..Hp-1 zero
  int H, Hp;
  float eps, gain;
  const float* part;      // n_part blocks [T, Hp] of partial sums still to be added to x, in order
  int n_part;
  size_t part_stride;
  const float* y;         // [T, Hp] branch: x += y / rms(y) * yw
  const elt* yw;          // [Hp]
  elt* out_frag;          // the normed row in fragment order (16-bit element types) ...
  int frag_tt;
  elt* out_row;           // ... and / or row-major [T, Hp]
  int raw;                // the output is x itself, rounded to the element type
};

// x += parts; x += y / rms(y) * yw; out = x / rms(x) * gain (or x).  One workgroup per row, the row in registers.
template <int VPT>
__global__ __launch_bounds__(SN_THREADS) void stream_norm_kernel(StreamNorm a) {
  __shared__ float lds[2][SN_THREADS / WAVE];
  const int row = blockIdx.x;
  float* xr = a.x + (size_t)row * a.Hp;
  f32x4 v[VPT];
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = (threadIdx.x + i * SN_THREADS) * 4;
    v[i] = c < a.Hp ? *reinterpret_cast<const f32x4*>(xr + c) : f32x4{0.f, 0.f, 0.f, 0.f};
  }
  for (int q = 0; q < a.n_part; ++q) {
    const float* pr = a.part + q * a.part_stride + (size_t)row * a.Hp;
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int c = (threadIdx.x + i * SN_THREADS) * 4;
      if (c < a.Hp) v[i] += *reinterpret_cast<const f32x4*>(pr + c);
    }
  }
  if (a.y) {
    const float* yr = a.y + (size_t)row * a.Hp;
    f32x4 b[VPT];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int c = (threadIdx.x + i * SN_THREADS) * 4;
      b[i] = c < a.Hp ? *reinterpret_cast<const f32x4*>(yr + c) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int e = 0; e < 4; ++e) ss = fmaf(b[i][e], b[i][e], ss);
    }
    const float inv = 1.f / sqrtf(sn_block_sum(ss, lds[0]) / (float)a.H + a.eps);
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int c = (threadIdx.x + i * SN_THREADS) * 4;
      if (c < a.Hp) {
        const eltx4 w = *reinterpret_cast<const eltx4*>(a.yw + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[i][e] += b[i][e] * inv * (float)w[e];
      }
    }
  }
  if (a.y || a.n_part) {
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int c = (threadIdx.x + i * SN_THREADS) * 4;
      if (c < a.Hp) *reinterpret_cast<f32x4*>(xr + c) = v[i];
    }
  }
  if (!a.out_frag && !a.out_row) return;
  float s = 1.f;
  if (!a.raw) {
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < VPT; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) ss = fmaf(v[i][e], v[i][e], ss);
    s = a.gain / sqrtf(sn_block_sum(ss, lds[1]) / (float)a.H + a.eps);
  }
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int c = (threadIdx.x + i * SN_THREADS) * 4;
    if (c >= a.Hp) continue;
    eltx4 o;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = (elt)(v[i][e] * s);
    if (a.out_frag) *reinterpret_cast<eltx4*>(a.out_frag + frag_offset(row, c, a.frag_tt)) = o;
    if (a.out_row) *reinterpret_cast<eltx4*>(a.out_row + (size_t)row * a.Hp + c) = o;
  }
}

__device__ __forceinline__ float gelu_tanh(float z) {
  return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

#ifndef MLORA_ELT_F32
// What becomes of four rows n .. n + 3 of a token's narrow product s = W x:
//   token gate: out[t, n] = gelu(s) * table[id_t, col0 + n] for n < dim, 0 for the padding rows, in fragment order
struct TokenGate {
  elt* out;
  const elt* table;
  int ld_table, col0, dim;
  const int32_t* ids;
  int V;
  __device__ __forceinline__ void operator()(int t, int n, f32x4 s, int frag_tt) const {
    const int id = ids[t];
    const bool ok = id >= 0 && id < V;
    eltx4 o;
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const float ev = ok && n + q < dim ? (float)table[(size_t)id * ld_table + col0 + n + q] : 0.f;
      o[q] = (elt)(gelu_tanh(s[q]) * ev);
    }
    *reinterpret_cast<eltx4*>(out + frag_offset(t, n, frag_tt)) = o;
  }
};
//   s itself, out [T][N] fp32
struct PlainRows {
  float* out;
  int N;
  __device__ __forceinline__ void operator()(int t, int n, f32x4 s, int) const { *reinterpret_cast<f32x4*>(out + (size_t)t * N + n) = s; }
};
//   tanh(s) in full precision as the sum of three elements, out [T][3][N]
struct TanhParts {
  elt* out;
  int N;
  __device__ __forceinline__ void operator()(int t, int n, f32x4 s, int) const {
    eltx4 o[3];
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      float v = tanhf(s[q]);
#pragma unroll
      for (int p = 0; p < 3; ++p) {
        o[p][q] = (elt)v;
        v -= (float)o[p][q];
      }
    }
#pragma unroll
    for (int p = 0; p < 3; ++p) *reinterpret_cast<eltx4*>(out + ((size_t)t * 3 + p) * N + n) = o[p];
  }
};

// The narrow product of a token block: x in fragment order, W packed.  A workgroup takes 16 TT tokens x 16 NT rows, its waves split
// K; a wave requests TG_U k-steps at a time.
constexpr int TG_WAVES = 8;
template <int NT, int TT, int TG_U, typename END>
__global__ __launch_bounds__(TG_WAVES* WAVE, 2) void token_gate_kernel(END end, int frag_tt, const elt* __restrict__ x, const elt* __restrict__ Wp, int T,
                                                                      int K, int N) {
  __shared__ f32x4 red[TG_WAVES][NT][WAVE];
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int KB = K / 32, tiles = N / 16;
  const int nt0 = blockIdx.x * NT, tt0 = blockIdx.y * TT;
  const elt* xp[TT];
#pragma unroll
  for (int j = 0; j < TT; ++j) xp[j] = x + (size_t)(tt0 + j < frag_tt ? tt0 + j : frag_tt - 1) * 512 + lane * 8;
  const elt* wp[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) wp[i] = Wp + (size_t)(nt0 + i < tiles ? nt0 + i : tiles - 1) * KB * 512 + lane * 8;
  f32x4 acc[NT][TT];
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int j = 0; j < TT; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int ks0 = wave; ks0 < KB; ks0 += TG_WAVES * TG_U) {
    eltx8 a[TG_U][NT], b[TG_U][TT];
#pragma unroll
    for (int u = 0; u < TG_U; ++u) {
      const bool in = ks0 + u * TG_WAVES < KB;                       // uniform; past K: a valid address, zeroed
      const int ks = in ? ks0 + u * TG_WAVES : ks0;
#pragma unroll
      for (int i = 0; i < NT; ++i) a[u][i] = ld8(wp[i] + (size_t)ks * 512);
#pragma unroll
      for (int j = 0; j < TT; ++j) {
        b[u][j] = ld8(xp[j] + (size_t)ks * frag_tt * 512);
        if (!in) b[u][j] = eltx8{0, 0, 0, 0, 0, 0, 0, 0};
      }
    }
#pragma unroll
    for (int u = 0; u < TG_U; ++u)
#pragma unroll
      for (int i = 0; i < NT; ++i)
#pragma unroll
        for (int j = 0; j < TT; ++j) acc[i][j] = mfma_16x16x32(a[u][i], b[u][j], acc[i][j]);
  }
#pragma unroll
  for (int j = 0; j < TT; ++j) {
    if (j > 0) __syncthreads();
#pragma unroll
    for (int i = 0; i < NT; ++i) red[wave][i][lane] = acc[i][j];
    __syncthreads();
    for (int e = threadIdx.x; e < NT * WAVE; e += TG_WAVES * WAVE) {
      const int i = e >> 6, sl = e & 63;
      const int t = (tt0 + j) * 16 + (sl & 15), n = (nt0 + i) * 16 + (sl >> 4) * 4;
      if (t >= T || n >= N) continue;
      f32x4 s = red[0][i][sl];
#pragma unroll
      for (int w = 1; w < TG_WAVES; ++w) s += red[w][i][sl];
      end(t, n, s, frag_tt);
    }
  }
}

template <typename END>
void launch_narrow(const END& end, const void* xf, const void* Wp, int T, int K, int N, hipStream_t s) {
#define MLORA_TG(NT, TT, U)                                                                                                                    \
  hipLaunchKernelGGL((token_gate_kernel<NT, TT, U, END>), dim3(ceil_div(N, 16 * NT), ceil_div(T, 16 * TT)), dim3(TG_WAVES * WAVE), 0, s, end, \
                     mlora_frag_tiles(T), (const elt*)xf, (const elt*)Wp, T, K, N)
  if (T <= 256) MLORA_TG(1, 1, 4);
  else if (N <= 32) MLORA_TG(2, 1, 4);
  else if ((long)ceil_div(N, 64) * ceil_div(T, 64) >= 256) MLORA_TG(4, 4, 2);      // a workgroup per compute unit with four token tiles
  else MLORA_TG(4, 1, 4);
#undef MLORA_TG
}
#endif

// the same product behind a separate linear: out[t, n] = gelu(z[t, n]) * table[id_t, col0 + n], row-major
__global__ __launch_bounds__(256) void token_gate_mul_kernel(elt* __restrict__ out, const elt* __restrict__ z, const elt* __restrict__ table,
                                                             int ld_table, int col0, int dim, const int32_t* __restrict__ ids, int V, int T, int N) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= (size_t)T * N) return;
  const int t = (int)(i / N), n = (int)(i % N);
  const int id = ids[t];
  const float ev = id >= 0 && id < V && n < dim ? (float)table[(size_t)id * ld_table + col0 + n] : 0.f;
  out[i] = (elt)(gelu_tanh((float)z[i]) * ev);
}

// ---------------------------------------------------------------------------------------------
// The residual stream of a decoder whose norms are elementwise, dt(v) = tanh(alpha v) w + b:
//   x' = x + mult post(branch),  branch = y + parts + row_weight * (entry rows of the token)
//   h  = pre(x'), written once, or as the mixes h + (h_prev - h) mu_s of a token and the one before it in its sequence
// No row statistics are needed, so the previous token's h is computed again instead of being exchanged.
// ---------------------------------------------------------------------------------------------
__device__ __forceinline__ f32x4 ld4f(const elt* p) {
  const eltx4 v = *reinterpret_cast<const eltx4*>(p);
  return f32x4{(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
}

// tanh to fp32 accuracy on the fast reciprocal and exponential: 1 - 2 / (exp(2 |x|) + 1), and its series where that cancels
__device__ __forceinline__ float tanh_f(float x) {
#ifdef MLORA_ELT_F32
  return tanhf(x);
#else
  const float a = fabsf(x), x2 = x * x;
  const float big = fmaf(-2.f, __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(a * 2.88539008177792681472f)), 1.f);
  const float small = fmaf(x2 * x, fmaf(x2, fmaf(x2, fmaf(x2, 62.f / 2835.f, -17.f / 315.f), 2.f / 15.f), -1.f / 3.f), x);
  return a < 0.25f ? small : copysignf(big, x);
#endif
}

struct TanhNorm {
  f32x4 w, b;
  float alpha;
  bool on;
  __device__ __forceinline__ TanhNorm(const mlora_tanh_norm& n, int c) : alpha(n.alpha), on(n.w != nullptr) {
    w = on ? ld4f((const elt*)n.w + c) : f32x4{1.f, 1.f, 1.f, 1.f};
    b = on ? ld4f((const elt*)n.b + c) : f32x4{0.f, 0.f, 0.f, 0.f};
  }
  __device__ __forceinline__ f32x4 operator()(f32x4 v) const {
    if (!on) return v;
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = fmaf(tanh_f(alpha * v[e]), w[e], b[e]);
    return v;
  }
};

// one token's four columns of x + mult post(branch)
__device__ __forceinline__ f32x4 step_row(const mlora_stream_step_args& a, const TanhNorm& post, int t, int c) {
  const size_t o = (size_t)t * a.Hp + c;
  f32x4 x = a.x ? *reinterpret_cast<const f32x4*>(a.x + o) : f32x4{0.f, 0.f, 0.f, 0.f};
  if (!a.y && !a.rows) return x;
  f32x4 v = a.y ? *reinterpret_cast<const f32x4*>(a.y + o) : f32x4{0.f, 0.f, 0.f, 0.f};
  for (int q = 0; q < a.n_part; ++q) v += *reinterpret_cast<const f32x4*>(a.part + (size_t)q * a.T * a.Hp + o);
  if (a.rows) {
    f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < a.top; ++k) s += ld4f((const elt*)a.rows + ((size_t)t * a.top + k) * a.Hp + c);
    v += s * a.row_weight;
  }
  v = post(v);
#pragma unroll
  for (int e = 0; e < 4; ++e) x[e] = fmaf(a.mult, v[e], x[e]);
  return x;
}

constexpr int ST_THREADS = 128;
constexpr int ST_MIX = 5;
// A thread takes four columns of `rows` consecutive tokens.
template <bool SHIFT>
__global__ __launch_bounds__(ST_THREADS) void stream_step_kernel(mlora_stream_step_args a, int rows, int frag_tt) {
  const int c = (blockIdx.x * ST_THREADS + threadIdx.x) * 4;
  if (c >= a.Hp) return;
  const TanhNorm post(a.post, c), pre(a.pre, c);
  const bool out = a.out_frag || a.out_row;
  f32x4 mu[SHIFT ? ST_MIX : 1], prev = f32x4{0.f, 0.f, 0.f, 0.f};
  int prev_seq = -1;                                                 // whose h `prev` is
  if constexpr (SHIFT) {
#pragma unroll
    for (int s = 0; s < ST_MIX; ++s) mu[s] = ld4f((const elt*)a.mu + (size_t)s * a.Hp + c);
  }
  const int t0 = blockIdx.y * rows, t1 = t0 + rows < a.T ? t0 + rows : a.T;
  for (int t = t0; t < t1; ++t) {
    const f32x4 x = step_row(a, post, t, c);
    if (a.x_out) *reinterpret_cast<f32x4*>(a.x_out + (size_t)t * a.Hp + c) = x;
    if (!out) continue;
    const f32x4 h = pre(x);
    if constexpr (SHIFT) {
      const int seq = a.tok_seq[t], pos = a.tok_pos[t];
      const bool live = seq >= 0 && seq < a.n_seq;
      if (pos <= 0) prev = f32x4{0.f, 0.f, 0.f, 0.f};
      else if (t > 0 && a.tok_seq[t - 1] == seq) {
        if (prev_seq < 0) prev = pre(step_row(a, post, t - 1, c));   // the token before belongs to another workgroup
      } else prev = live ? *reinterpret_cast<const f32x4*>(a.shift + (size_t)seq * a.Hp + c) : f32x4{0.f, 0.f, 0.f, 0.f};
      if (live && (t == 0 || a.tok_seq[t - 1] != seq)) {
        // the sequence's first token of the pass read the state; it also leaves the last one's h there
        int last = a.tok_last ? a.tok_last[t] : t;
        last = last < a.T ? last : a.T - 1;
        *reinterpret_cast<f32x4*>(a.shift + (size_t)seq * a.Hp + c) = last > t ? pre(step_row(a, post, last, c)) : h;
      }
#pragma unroll
      for (int s = 0; s < ST_MIX; ++s) {
        eltx4 o;
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = (elt)fmaf(prev[e] - h[e], mu[s][e], h[e]);
        if (a.out_frag) *reinterpret_cast<eltx4*>((elt*)a.out_frag + s * (size_t)a.mix_stride + frag_offset(t, c, frag_tt)) = o;
        if (a.out_row) *reinterpret_cast<eltx4*>((elt*)a.out_row + s * (size_t)a.mix_stride + (size_t)t * a.ld_row + c) = o;
      }
      prev = h;
      prev_seq = 0;
    } else {
      const eltx4 o = eltx4{(elt)h[0], (elt)h[1], (elt)h[2], (elt)h[3]};
      if (a.out_frag) *reinterpret_cast<eltx4*>((elt*)a.out_frag + frag_offset(t, c, frag_tt)) = o;
      if (a.out_row) *reinterpret_cast<eltx4*>((elt*)a.out_row + (size_t)t * a.ld_row + c) = o;
    }
  }
}

#ifndef MLORA_ELT_F32
struct F8 {
  f32x4 v[2];
};
__device__ __forceinline__ F8 ld8f(const float* p) { return F8{{*reinterpret_cast<const f32x4*>(p), *reinterpret_cast<const f32x4*>(p + 4)}}; }
struct TanhNorm8 {          // weights as elements: they stay in registers over many tokens
  eltx8 w, b;
  float alpha;
  bool on;
  __device__ __forceinline__ TanhNorm8(const mlora_tanh_norm& n, int c) : alpha(n.alpha), on(n.w != nullptr) {
    w = b = eltx8{0, 0, 0, 0, 0, 0, 0, 0};
    if (on) {
      w = ld8((const elt*)n.w + c);
      b = ld8((const elt*)n.b + c);
    }
  }
  __device__ __forceinline__ F8 operator()(F8 x) const {
    if (!on) return x;                                               // uniform
#pragma unroll
    for (int e = 0; e < 8; ++e) x.v[e >> 2][e & 3] = fmaf(tanh_f(alpha * x.v[e >> 2][e & 3]), (float)w[e], (float)b[e]);
    return x;
  }
};

// one token's eight columns of x + mult post(branch)
__device__ __forceinline__ F8 step_row8(const mlora_stream_step_args& a, const TanhNorm8& post, int t, int c) {
  const size_t o = (size_t)t * a.Hp + c;
  F8 x = F8{{f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}}}, v = x;
  if (a.x) x = ld8f(a.x + o);
  if (!a.y && !a.rows) return x;
  if (a.y) v = ld8f(a.y + o);
  for (int q = 0; q < a.n_part; ++q) {
    const F8 p = ld8f(a.part + (size_t)q * a.T * a.Hp + o);
    v.v[0] += p.v[0];
    v.v[1] += p.v[1];
  }
  if (a.rows) {
    const elt* rp = (const elt*)a.rows + (size_t)t * a.top * a.Hp + c;
    F8 s = F8{{f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}}};
    for (int k0 = 0; k0 < a.top; k0 += 4) {                          // four rows are requested together
      eltx8 r[4];
#pragma unroll
      for (int k = 0; k < 4; ++k) r[k] = ld8(rp + (size_t)(k0 + k < a.top ? k0 + k : k0) * a.Hp);
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const float f = k0 + k < a.top ? 1.f : 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) s.v[e >> 2][e & 3] = fmaf(f, (float)r[k][e], s.v[e >> 2][e & 3]);
      }
    }
    v.v[0] += s.v[0] * a.row_weight;
    v.v[1] += s.v[1] * a.row_weight;
  }
  v = post(v);
#pragma unroll
  for (int e = 0; e < 8; ++e) x.v[e >> 2][e & 3] = fmaf(a.mult, v.v[e >> 2][e & 3], x.v[e >> 2][e & 3]);
  return x;
}

// The same with outputs in fragment order: a wave takes 32 columns of `tiles` tiles of 16 tokens - lane (token q16, columns
// 8 g ..) - so that it reads whole lines of the stream and writes whole fragments, and a token's neighbour is the lane beside it.
template <bool SHIFT>
__global__ __launch_bounds__(256) void stream_step_tile_kernel(mlora_stream_step_args a, int tiles, int frag_tt) {
  const int lane = threadIdx.x & 63, q16 = lane & 15, g = lane >> 4;
  const int ks = blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), c = ks * 32 + g * 8;
  if (ks * 32 >= a.Hp) return;                                       // uniform; no barrier below
  const TanhNorm8 post(a.post, c), pre(a.pre, c);
  eltx8 mu[SHIFT ? ST_MIX : 1];
  if constexpr (SHIFT) {
#pragma unroll
    for (int s = 0; s < ST_MIX; ++s) mu[s] = ld8((const elt*)a.mu + (size_t)s * a.Hp + c);
  }
  F8 carry = F8{{f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}}};      // the row ahead of the tile
  bool carried = false;                                              // uniform
  const int tile0 = blockIdx.y * tiles;
  for (int i = 0; i < tiles; ++i) {
    const int t0 = (tile0 + i) * 16, t = t0 + q16;
    if (t0 >= a.T) return;                                           // uniform
    const bool in = t < a.T;
    const int tc = in ? t : a.T - 1;
    const F8 x = step_row8(a, post, tc, c);
    if (a.x_out && in) {
      f32x4* p = reinterpret_cast<f32x4*>(a.x_out + (size_t)t * a.Hp + c);
      p[0] = x.v[0];
      p[1] = x.v[1];
    }
    const F8 h = pre(x);
    elt* fp = (elt*)a.out_frag + ((size_t)ks * frag_tt + tile0 + i) * 512 + g * 128 + q16 * 8;   // exists also for the tile's tokens behind T
    if constexpr (SHIFT) {
      const int seq = a.tok_seq[tc], pos = a.tok_pos[tc];
      const int seq_p = tc > 0 ? a.tok_seq[tc - 1] : -1;
      const bool live = in && seq >= 0 && seq < a.n_seq, cont = tc > 0 && seq_p == seq;
      F8 prev;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float p = row_shr<1>(h.v[e >> 2][e & 3]);
        prev.v[e >> 2][e & 3] = q16 > 0 ? p : carry.v[e >> 2][e & 3];
      }
      if (in && q16 == 0 && cont && pos > 0 && !carried) prev = pre(step_row8(a, post, t - 1, c));     // it belongs to another workgroup
      if (in && !cont && pos > 0) {
        prev = F8{{f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}}};
        if (live) prev = ld8f(a.shift + (size_t)seq * a.Hp + c);
      }
      if (pos <= 0) prev = F8{{f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}}};
      if (live && !cont) {
        // the sequence's first token of the pass read the state; it also leaves the last one's row there
        int last = a.tok_last ? a.tok_last[t] : t;
        last = last < a.T ? last : a.T - 1;
        const F8 l = last > t ? pre(step_row8(a, post, last, c)) : h;
        f32x4* p = reinterpret_cast<f32x4*>(a.shift + (size_t)seq * a.Hp + c);
        p[0] = l.v[0];
        p[1] = l.v[1];
      }
#pragma unroll
      for (int s = 0; s < ST_MIX; ++s) {
        eltx8 o;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float hv = h.v[e >> 2][e & 3];
          o[e] = (elt)fmaf(prev.v[e >> 2][e & 3] - hv, (float)mu[s][e], hv);
        }
        st8(fp + s * (size_t)a.mix_stride, o);
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) carry.v[e >> 2][e & 3] = row_lane<15>(h.v[e >> 2][e & 3]);
      carried = true;
    } else {
      eltx8 o;
#pragma unroll
      for (int e = 0; e < 8; ++e) o[e] = (elt)h.v[e >> 2][e & 3];
      st8(fp, o);
      if (a.out_row && in) st8((elt*)a.out_row + (size_t)t * a.ld_row + c, o);
    }
  }
}
#endif

// x = table[id] * scale in fp32, and the same rounded, in fragment order or with a row stride of its own
__global__ __launch_bounds__(256) void embed_scaled_kernel(float* __restrict__ x, elt* __restrict__ out_frag, int frag_tt, elt* __restrict__ out_row,
                                                           int ld_row, const elt* __restrict__ table, const int32_t* __restrict__ ids, float scale,
                                                           int H, int V) {
  const int t = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 4;
  if (c >= H) return;
  const int id = ids[t];
  f32x4 v = f32x4{0.f, 0.f, 0.f, 0.f};
  if (id >= 0 && id < V) v = ld4f(table + (size_t)id * H + c) * scale;
  *reinterpret_cast<f32x4*>(x + (size_t)t * H + c) = v;
  const eltx4 o = eltx4{(elt)v[0], (elt)v[1], (elt)v[2], (elt)v[3]};
  if (out_frag) *reinterpret_cast<eltx4*>(out_frag + frag_offset(t, c, frag_tt)) = o;
  if (out_row) *reinterpret_cast<eltx4*>(out_row + (size_t)t * ld_row + c) = o;
}

}  // namespace

extern "C" int mlora_stream_norm(void* out_frag, void* out_row, float* x, const float* part, int n_part, const float* branch,
                                 const void* branch_w, float eps, float gain, int raw, int T, int H, int Hp, void* stream) {
  MLORA_CHECK(x && T >= 0 && H > 0 && Hp >= H && Hp % 32 == 0 && Hp <= 16384, MLORA_ERR_UNSUPPORTED,
              "stream_norm: need 0 < H <= Hp <= 16384, Hp %% 32 == 0 (T=%d H=%d Hp=%d)", T, H, Hp);
  MLORA_CHECK((n_part == 0 || part) && n_part >= 0 && (!branch || branch_w), MLORA_ERR_INVALID, "stream_norm: null pointer");
  MLORA_CHECK(!out_frag || sizeof(elt) == 2, MLORA_ERR_UNSUPPORTED, "stream_norm: fragment order is for 16-bit elements");
  if (T == 0) return MLORA_OK;
  StreamNorm a;
  a.x = x; a.H = H; a.Hp = Hp; a.eps = eps; a.gain = gain;
  a.part = part; a.n_part = n_part; a.part_stride = (size_t)T * Hp;
  a.y = branch; a.yw = (const elt*)branch_w;
  a.out_frag = (elt*)out_frag; a.frag_tt = mlora_frag_tiles(T); a.out_row = (elt*)out_row; a.raw = raw;
  hipStream_t s = (hipStream_t)stream;
  if (Hp <= 2048) hipLaunchKernelGGL(stream_norm_kernel<2>, dim3(T), dim3(SN_THREADS), 0, s, a);
  else if (Hp <= 4096) hipLaunchKernelGGL(stream_norm_kernel<4>, dim3(T), dim3(SN_THREADS), 0, s, a);
  else if (Hp <= 8192) hipLaunchKernelGGL(stream_norm_kernel<8>, dim3(T), dim3(SN_THREADS), 0, s, a);
  else hipLaunchKernelGGL(stream_norm_kernel<16>, dim3(T), dim3(SN_THREADS), 0, s, a);
  return mlora_launch_status("stream_norm");
}

#ifndef MLORA_ELT_F32
extern "C" int mlora_token_gate(void* out_frag, const void* xf, const void* Wp, const void* table, int ld_table, int col0, int dim,
                                const int32_t* ids, int V, int T, int K, int N, void* stream) {
  MLORA_CHECK(out_frag && xf && Wp && table && ids, MLORA_ERR_INVALID, "token_gate: null pointer");
  MLORA_CHECK(T >= 0 && K > 0 && K % 32 == 0 && N > 0 && N % 32 == 0 && dim > 0 && dim <= N && col0 >= 0 && col0 + dim <= ld_table && V > 0 &&
                  ceil_div(T, 16) <= 65535,
              MLORA_ERR_UNSUPPORTED, "token_gate: need K %% 32 == 0, N %% 32 == 0, dim <= N (T=%d K=%d N=%d dim=%d)", T, K, N, dim);
  if (T == 0) return MLORA_OK;
  launch_narrow(TokenGate{(elt*)out_frag, (const elt*)table, ld_table, col0, dim, ids, V}, xf, Wp, T, K, N, (hipStream_t)stream);
  return mlora_launch_status("token_gate");
}

extern "C" int mlora_narrow_linear(float* out, const void* xf, const void* Wp, int T, int K, int N, void* stream) {
  MLORA_CHECK(out && xf && Wp, MLORA_ERR_INVALID, "narrow_linear: null pointer");
  MLORA_CHECK(T >= 0 && K > 0 && K % 32 == 0 && N > 0 && N % 32 == 0 && ceil_div(T, 16) <= 65535, MLORA_ERR_UNSUPPORTED,
              "narrow_linear: need K %% 32 == 0, N %% 32 == 0 (T=%d K=%d N=%d)", T, K, N);
  if (T == 0) return MLORA_OK;
  launch_narrow(PlainRows{out, N}, xf, Wp, T, K, N, (hipStream_t)stream);
  return mlora_launch_status("narrow_linear");
}

extern "C" int mlora_tanh_parts(void* out, const void* xf, const void* Wp, int T, int K, int N, void* stream) {
  MLORA_CHECK(out && xf && Wp, MLORA_ERR_INVALID, "tanh_parts: null pointer");
  MLORA_CHECK(T >= 0 && K > 0 && K % 32 == 0 && N > 0 && N % 32 == 0 && ceil_div(T, 16) <= 65535, MLORA_ERR_UNSUPPORTED,
              "tanh_parts: need K %% 32 == 0, N %% 32 == 0 (T=%d K=%d N=%d)", T, K, N);
  if (T == 0) return MLORA_OK;
  launch_narrow(TanhParts{(elt*)out, N}, xf, Wp, T, K, N, (hipStream_t)stream);
  return mlora_launch_status("tanh_parts");
}
#endif

extern "C" int mlora_token_gate_mul(void* out, const void* z, const void* table, int ld_table, int col0, int dim, const int32_t* ids, int V,
                                    int T, int N, void* stream) {
  MLORA_CHECK(out && z && table && ids, MLORA_ERR_INVALID, "token_gate_mul: null pointer");
  MLORA_CHECK(T >= 0 && N > 0 && dim > 0 && dim <= N && col0 >= 0 && col0 + dim <= ld_table && V > 0 && (size_t)T * N / 256 < 0x7fffffffULL,
              MLORA_ERR_UNSUPPORTED, "token_gate_mul: bad shape T=%d N=%d dim=%d", T, N, dim);
  if (T == 0) return MLORA_OK;
  hipLaunchKernelGGL(token_gate_mul_kernel, dim3((unsigned)(((size_t)T * N + 255) / 256)), dim3(256), 0, (hipStream_t)stream, (elt*)out,
                     (const elt*)z, (const elt*)table, ld_table, col0, dim, ids, V, T, N);
  return mlora_launch_status("token_gate_mul");
}

extern "C" int mlora_stream_step(const mlora_stream_step_args* args, void* stream) {
  MLORA_CHECK(args, MLORA_ERR_INVALID, "stream_step: null pointer");
  const mlora_stream_step_args& a = *args;
  MLORA_CHECK(a.T >= 0 && a.Hp > 0 && a.Hp % 32 == 0 && a.n_part >= 0 && a.T <= 65535 * 8, MLORA_ERR_UNSUPPORTED,
              "stream_step: need Hp %% 32 == 0 (T=%d Hp=%d)", a.T, a.Hp);
  MLORA_CHECK((a.x || a.y || a.rows) && (a.n_part == 0 || (a.part && a.y)) && (!a.rows || a.top > 0) && (!a.post.w || a.post.b) && (!a.pre.w || a.pre.b),
              MLORA_ERR_INVALID, "stream_step: null pointer");
  MLORA_CHECK(!a.out_frag || sizeof(elt) == 2, MLORA_ERR_UNSUPPORTED, "stream_step: fragment order is for 16-bit elements");
  MLORA_CHECK(!a.out_row || (a.ld_row >= a.Hp && a.ld_row % 4 == 0), MLORA_ERR_INVALID, "stream_step: row stride %d", a.ld_row);
  if (a.mu)
    MLORA_CHECK(a.shift && a.tok_seq && a.tok_pos && a.n_seq > 0 && (a.out_frag || a.out_row) && (!(a.y || a.rows) || a.x_out != a.x), MLORA_ERR_INVALID,
                "stream_step: the mixes need the state, the tokens' sequences and a stream that is not updated in place");
  if (a.T == 0) return MLORA_OK;
  hipStream_t s = (hipStream_t)stream;
  const int tt = mlora_frag_tiles(a.T);
#ifndef MLORA_ELT_F32
  if (a.out_frag && !(a.mu && a.out_row) && a.ld_row % 8 == 0) {
    const int cb = ceil_div(a.Hp, 128), nt = ceil_div(a.T, 16);
    int tiles = 1;
    while (tiles < 8 && (long)cb * ceil_div(nt, 2 * tiles) >= 1024) tiles *= 2;
    while (ceil_div(nt, tiles) > 65535) tiles *= 2;
    const dim3 grid(cb, ceil_div(nt, tiles));
    if (a.mu) hipLaunchKernelGGL(stream_step_tile_kernel<true>, grid, dim3(256), 0, s, a, tiles, tt);
    else hipLaunchKernelGGL(stream_step_tile_kernel<false>, grid, dim3(256), 0, s, a, tiles, tt);
    return mlora_launch_status("stream_step");
  }
#endif
  const int cols = ceil_div(a.Hp, ST_THREADS * 4);
  int rows = 1;
  while (rows < 8 && (long)cols * ceil_div(a.T, 2 * rows) >= 2048) rows *= 2;
  while (ceil_div(a.T, rows) > 65535) rows *= 2;
  const dim3 grid(cols, ceil_div(a.T, rows));
  if (a.mu) hipLaunchKernelGGL(stream_step_kernel<true>, grid, dim3(ST_THREADS), 0, s, a, rows, tt);
  else hipLaunchKernelGGL(stream_step_kernel<false>, grid, dim3(ST_THREADS), 0, s, a, rows, tt);
  return mlora_launch_status("stream_step");
}

extern "C" int mlora_embed_scaled(float* x, void* out_frag, void* out_row, int ld_row, const void* table, const int32_t* ids, float scale, int T, int H,
                                  int V, void* stream) {
  MLORA_CHECK(x && table && ids, MLORA_ERR_INVALID, "embed_scaled: null pointer");
  MLORA_CHECK(T >= 0 && T <= 65535 && H > 0 && H % 32 == 0 && V > 0 && (!out_frag || sizeof(elt) == 2) && (!out_row || (ld_row >= H && ld_row % 4 == 0)),
              MLORA_ERR_UNSUPPORTED, "embed_scaled: need H %% 32 == 0 (T=%d H=%d V=%d)", T, H, V);
  if (T == 0) return MLORA_OK;
  hipLaunchKernelGGL(embed_scaled_kernel, dim3(ceil_div(H, 1024), T), dim3(256), 0, (hipStream_t)stream, x, (elt*)out_frag, mlora_frag_tiles(T),
                     (elt*)out_row, ld_row, (const elt*)table, ids, scale, H, V);
  return mlora_launch_status("embed_scaled");
}
