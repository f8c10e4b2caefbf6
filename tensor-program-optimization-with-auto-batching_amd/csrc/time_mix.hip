// Time mixing with a matrix state per head and a decay per key channel (a linear recurrence):
//     o_t = (S + diag(u) k_t v_t^T)^T r_t        S <- diag(w_t) S + k_t v_t^T
//     w_t = exp(-exp(W2 tanh(z_t) + w0))         z_t: the decay's low-rank projection of the token
//     y_t = o_t / rms(o_t) * norm * silu(g_t)    rms over the head
// r, k, v, g [T, ld] in elements (columns head * D + channel), z [T, ld_z] fp32; everything behind the projections is fp32.
// The state [n_seq, H, D (key), D (value)] fp32 belongs to a sequence's slot; a sequence whose first token of the pass has
// position 0 starts from zero, whatever the slot holds.  Compiled for every element type.
//
// Three forms of the same sums: token by token (time_mix_scan_kernel), one token per sequence (time_mix_step_kernel) and, in the
// bfloat16 library, chunks of 16 tokens on the matrix cores (time_mix_chunk_kernel).
#include <type_traits>

#include "common.h"

namespace {

struct TimeMix {
  elt* y;                   // row-major [T, ld_y] or (frag_tt > 0) fragment order
  int frag_tt, ld_y;
  const elt* r;
  const elt* k;
  const elt* v;
  const elt* g;
  int ld;
  const float* z;           // [n_z, T, ld_z] partial sums, R columns count
  int n_z, ld_z, R;
  const elt* w2;            // [H * D, ld_w2], zero behind the R columns
  int ld_w2;
  const float* w0;          // [H * D]
  const float* u;           // [H * D]
  const elt* norm;          // [H * D]
  float eps;
  float* state;
  int n_seq, H, D, T;
  const int4* segs;         // {slot, first token, tokens, position of the first}; nullptr: every token is a sequence of its own
  const int32_t* tok_seq;
  const int32_t* tok_pos;
};

__device__ __forceinline__ float rank_tanh(const TimeMix& a, int t, int j) {
  if (j >= a.R) return 0.f;
  float z = 0.f;
  for (int q = 0; q < a.n_z; ++q) z += a.z[((size_t)q * a.T + t) * a.ld_z + j];
  return tanhf(z);
}

__device__ __forceinline__ int4 segment(const TimeMix& a, int i) {
  if (a.segs) return a.segs[i];
  return make_int4(a.tok_seq[i], i, 1, a.tok_pos[i]);
}

constexpr int TM_MAX_R = 256;
// A workgroup runs one head of one sequence token by token: C columns of the state (values) x KG groups of ROWS rows (keys)
// over its threads, the state in registers.  CH tokens at a time: inputs and decays go to LDS, the groups' partial sums
// meet there, then a wave per token norms and gates.
template <int ROWS, int C, int KG, int CH>
__global__ __launch_bounds__(C* KG) void time_mix_scan_kernel(TimeMix a) {
  constexpr int NT = C * KG, NW = NT / WAVE;
  constexpr int DM = ROWS * KG < C ? C : ROWS * KG;                  // rows of the buffers (>= D)
  __shared__ __align__(16) float rs[CH][DM], ks[CH][DM], ws[CH][DM], vs[CH][C], op[KG][CH][C];
  __shared__ float zs[CH][TM_MAX_R];
  const int h = blockIdx.x, D = a.D, hd = h * D;
  const int4 seg = segment(a, blockIdx.y);
  if (seg.x < 0 || seg.x >= a.n_seq || seg.z <= 0) return;           // uniform
  const int c = threadIdx.x % C, kg = threadIdx.x / C;               // a wave lies inside one group (C is a multiple of 64)
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  float* sp = a.state + ((size_t)seg.x * a.H + h) * D * D;
  float S[ROWS], uu[ROWS];
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int row = kg * ROWS + i;
    S[i] = seg.w > 0 && row < D && c < D ? sp[(size_t)row * D + c] : 0.f;
    uu[i] = row < D ? a.u[hd + row] : 0.f;
  }
  for (int n0 = 0; n0 < seg.z; n0 += CH) {
    const int n = seg.z - n0 < CH ? seg.z - n0 : CH;
    const int tb = seg.y + n0;
    __syncthreads();
    for (int i = threadIdx.x; i < n * a.ld_w2; i += NT) {
      const int t = i / a.ld_w2, j = i - t * a.ld_w2;
      zs[t][j] = rank_tanh(a, tb + t, j);
    }
    for (int i = threadIdx.x; i < n * DM; i += NT) {
      const int t = i / DM, d = i - t * DM;
      const size_t o = (size_t)(tb + t) * a.ld + hd + d;
      const bool in = d < D;
      rs[t][d] = in ? (float)a.r[o] : 0.f;
      ks[t][d] = in ? (float)a.k[o] : 0.f;
      if (d < C) vs[t][d] = in ? (float)a.v[o] : 0.f;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < n * DM; i += NT) {
      const int t = i / DM, d = i - t * DM;
      float w = 0.f;
      if (d < D) {
        float s = a.w0[hd + d];
        for (int j = 0; j < a.ld_w2; j += 8) {
          const eltx8 v = ld8(a.w2 + (size_t)(hd + d) * a.ld_w2 + j);
#pragma unroll
          for (int e = 0; e < 8; ++e) s = fmaf(zs[t][j + e], (float)v[e], s);
        }
        w = expf(-expf(s));
      }
      ws[t][d] = w;
    }
    __syncthreads();
    for (int t = 0; t < n; ++t) {
      const float vv = vs[t][c];
      float o = 0.f;
#pragma unroll
      for (int i = 0; i < ROWS; i += 4) {
        const f32x4 r4 = *reinterpret_cast<const f32x4*>(&rs[t][kg * ROWS + i]), k4 = *reinterpret_cast<const f32x4*>(&ks[t][kg * ROWS + i]),
                    w4 = *reinterpret_cast<const f32x4*>(&ws[t][kg * ROWS + i]);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float kv = k4[e] * vv;
          o = fmaf(r4[e], fmaf(uu[i + e], kv, S[i + e]), o);
          S[i + e] = fmaf(w4[e], S[i + e], kv);
        }
      }
      op[kg][t][c] = o;
    }
    __syncthreads();
    for (int t = wave; t < n; t += NW) {                             // a wave per token
      float o[C / WAVE], ss = 0.f;
#pragma unroll
      for (int q = 0; q < C / WAVE; ++q) {
        const int d = q * WAVE + lane;
        float s = op[0][t][d];
#pragma unroll
        for (int e = 1; e < KG; ++e) s += op[e][t][d];
        o[q] = s;
        ss = fmaf(s, s, ss);                                         // columns behind D are zero
      }
      const float inv = 1.f / sqrtf(wave_sum(ss) / (float)D + a.eps);
      const int tt = tb + t;
#pragma unroll
      for (int q = 0; q < C / WAVE; ++q) {
        const int d = q * WAVE + lane;
        if (d >= D) continue;
        const float g = (float)a.g[(size_t)tt * a.ld + hd + d];
        const float v = o[q] * inv * (float)a.norm[hd + d] * (g / (1.f + expf(-g)));
        a.y[a.frag_tt ? frag_offset(tt, hd + d, a.frag_tt) : (size_t)tt * a.ld_y + hd + d] = (elt)v;
      }
    }
  }
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int row = kg * ROWS + i;
    if (row < D && c < D) sp[(size_t)row * D + c] = S[i];
  }
}

constexpr int TS_THREADS = 256;
// A decode step: one workgroup per (token, head).  A thread takes four columns (values) of every RG-th row (key); the whole state is
// requested before anything else.  C: columns of the buffers (D <= C), a power of two up to 128.
template <int C>
__global__ __launch_bounds__(TS_THREADS) void time_mix_step_kernel(TimeMix a) {
  constexpr int CG = C / 4, RG = TS_THREADS / CG, ROWS = C / RG;     // column groups, row groups, rows per thread
  constexpr int DP = TS_THREADS / C;                                 // threads that share a channel's decay
  __shared__ __align__(16) float zs[TM_MAX_R], rk[C], ks[C], ws[C], us[C], op[TS_THREADS / WAVE][C];
  __shared__ float red[2];
  const int h = blockIdx.x, D = a.D, hd = h * D, t = blockIdx.y;
  const int seq = a.tok_seq[t], pos = a.tok_pos[t];
  if (seq < 0 || seq >= a.n_seq) return;                             // uniform
  const int c = (threadIdx.x % CG) * 4, rg = threadIdx.x / CG;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  float* sp = a.state + ((size_t)seq * a.H + h) * D * D;
  const bool whole = D == C;                                         // uniform: rows are 16-byte aligned and need no bounds
  f32x4 S[ROWS];
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int row = i * RG + rg;
    S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (pos <= 0) continue;                                          // uniform
    if (whole) {
      S[i] = *reinterpret_cast<const f32x4*>(sp + (size_t)row * D + c);
    } else if (row < D) {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (c + e < D) S[i][e] = sp[(size_t)row * D + c + e];
    }
  }
  const size_t o0 = (size_t)t * a.ld + hd;
  f32x4 v4 = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int e = 0; e < 4; ++e)
    if (c + e < D) v4[e] = (float)a.v[o0 + c + e];
  for (int j = threadIdx.x; j < a.ld_w2; j += TS_THREADS) zs[j] = rank_tanh(a, t, j);
  if (threadIdx.x < C) {
    const int d = threadIdx.x;
    rk[d] = d < D ? (float)a.r[o0 + d] : 0.f;
    ks[d] = d < D ? (float)a.k[o0 + d] : 0.f;
    us[d] = d < D ? a.u[hd + d] : 0.f;
  }
  __syncthreads();
  {
    const int d = threadIdx.x / DP, q = threadIdx.x % DP;            // consecutive threads share a channel
    float s = 0.f;
    if (d < D)
      for (int j = q * 8; j < a.ld_w2; j += DP * 8) {
        const eltx8 v = ld8(a.w2 + (size_t)(hd + d) * a.ld_w2 + j);
#pragma unroll
        for (int e = 0; e < 8; ++e) s = fmaf(zs[j + e], (float)v[e], s);
      }
#pragma unroll
    for (int o = DP / 2; o > 0; o >>= 1) s += __shfl_xor(s, o, WAVE);
    if (q == 0) ws[d] = d < D ? expf(-expf(s + a.w0[hd + d])) : 0.f;
  }
  __syncthreads();
  f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int row = i * RG + rg;
    const f32x4 kv = v4 * ks[row];
    const float r = rk[row], u = us[row], w = ws[row];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      o[e] = fmaf(r, fmaf(u, kv[e], S[i][e]), o[e]);
      S[i][e] = fmaf(w, S[i][e], kv[e]);
    }
    if (whole) {
      *reinterpret_cast<f32x4*>(sp + (size_t)row * D + c) = S[i];
    } else if (row < D) {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (c + e < D) sp[(size_t)row * D + c + e] = S[i][e];
    }
  }
#pragma unroll
  for (int q = CG; q < WAVE; q <<= 1)
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] += __shfl_xor(o[e], q, WAVE);
  if (lane < CG) *reinterpret_cast<f32x4*>(&op[wave][c]) = o;
  __syncthreads();
  float x = 0.f;
  if (threadIdx.x < C) {
#pragma unroll
    for (int w = 0; w < TS_THREADS / WAVE; ++w) x += op[w][threadIdx.x];
  }
  const float ss = wave_sum(x * x);                                  // columns behind the head are zero
  if (lane == 0 && wave < 2) red[wave] = ss;
  __syncthreads();
  const int d = threadIdx.x;
  if (d < D) {
    const float inv = 1.f / sqrtf((red[0] + red[1]) / (float)D + a.eps);
    const float g = (float)a.g[o0 + d];
    a.y[a.frag_tt ? frag_offset(t, hd + d, a.frag_tt) : (size_t)t * a.ld_y + hd + d] = (elt)(x * inv * (float)a.norm[hd + d] * (g / (1.f + expf(-g))));
  }
}

#ifndef MLORA_ELT_F32
// ---------------------------------------------------------------------------------------------
// Chunks of 16 tokens.  With L_t the sum of the logarithms of the decays of a chunk's tokens up to t (Lx_t: without t's own),
//   o_t = (r_t exp Lx_t)^T S + sum_(s < t) A_ts v_s + (r_t . u k_t) v_t       A_ts = sum_d r_t k_s exp(Lx_t - L_s)
//   S  <- diag(exp L_15) S + sum_s (k_s exp(L_15 - L_s)) v_s^T
// A is made of products whose factors are all at most one: two tokens that part at bit h of their number meet at the last
// token m of the lower half of their block of 2 h, exp(Lx_t - L_m) exp(L_m - L_s).  At every level h = 8, 4, 2, 1 a token is in one
// half, so one vector x per token and level holds r's factor or k's, and the level's part of A is a part of x x^T.  Decays of any
// strength are served; nothing overflows.
// fp32 operands of the matrix cores are hi + lo pairs (what enters the state has a third part, and values are elements, so that the
// state is summed in fp32), in the two halves of the 32 k-slots: slot (g, e) is index 4 g + e for e < 4 as hi (or of the one factor)
// and again for e >= 4 as lo.  That is also how a lane holds a result (rows 4 g + r), so a
// state tile is an operand as it stands, and a product with the identity turns a factor over.
//
// A workgroup takes one head and up to a range of `tokens` of a sequence; wave w holds keys 16 w .. + 15 of the state (all values) and
// finishes values 16 w .. + 15 of the outputs.  Ranges of a sequence run side by side: a first launch (OUT false) leaves what a range
// adds to the state, time_mix_range_kernel makes the state ahead of every range of it.
// ---------------------------------------------------------------------------------------------
struct TimeMixRange {       // 8 int32
  int slot, first, tokens, pos;      // pos: of the range's first token
  int in;                   // scratch state the range starts from, -1: the slot's (zero at position 0)
  int add;                  // scratch state that takes what the range adds (first launch), -1: none
  int last;                 // the sequence's last range of the pass: leaves its state in the slot
  int pad;
};

__device__ __forceinline__ float quad_lane1(float v) {               // lane 1's of the 4
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x55, 0xf, 0xf, false));
}

// four floats as pairs of elements hi + lo (each word two elements)
struct HiLo {
  uint32_t h[2], l[2];
  __device__ __forceinline__ HiLo(f32x4 v) {
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      h[i] = __builtin_bit_cast(uint32_t, __builtin_convertvector((f32x2{v[2 * i], v[2 * i + 1]}), eltx2));
      const f32x2 rest = f32x2{v[2 * i] - __uint_as_float(h[i] << 16), v[2 * i + 1] - __uint_as_float(h[i] & 0xffff0000u)};
      l[i] = __builtin_bit_cast(uint32_t, __builtin_convertvector(rest, eltx2));
    }
  }
};
typedef uint32_t u32x2 __attribute__((ext_vector_type(2)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
__device__ __forceinline__ eltx8 operand(uint32_t a, uint32_t b, uint32_t c, uint32_t d) { return __builtin_bit_cast(eltx8, (u32x4{a, b, c, d})); }
__device__ __forceinline__ eltx8 both(const HiLo& v) { return operand(v.h[0], v.h[1], v.l[0], v.l[1]); }
// (a, b) and its halves swapped: two products with a pair of pairs make all four of their parts
__device__ __forceinline__ eltx8 swapped(const HiLo& v) { return operand(v.l[0], v.l[1], v.h[0], v.h[1]); }
__device__ __forceinline__ f32x4 floats(u32x2 v) {
  return f32x4{__uint_as_float(v[0] << 16), __uint_as_float(v[0] & 0xffff0000u), __uint_as_float(v[1] << 16), __uint_as_float(v[1] & 0xffff0000u)};
}
__device__ __forceinline__ f32x4 exp2_4(f32x4 v) {
  return f32x4{__builtin_amdgcn_exp2f(v[0]), __builtin_amdgcn_exp2f(v[1]), __builtin_amdgcn_exp2f(v[2]), __builtin_amdgcn_exp2f(v[3])};
}
// LDS accesses done, then the bare barrier: the next chunk's requests stay in flight
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  bare_barrier();
}

constexpr int TC_RK = 2;       // k-steps of the decay's rank whose weights stay in registers
// NT: 16-channel tiles of a head and waves; FULL: the head has exactly so many channels; OUT: see above
template <int NT, bool FULL, bool OUT>
__global__ __launch_bounds__(NT * WAVE, 2) void time_mix_chunk_kernel(TimeMix a, const elt* __restrict__ zp, int rb, const TimeMixRange* __restrict__ ranges,
                                                                    float* __restrict__ scratch, float* __restrict__ decay) {
  extern __shared__ __align__(16) char smem[];
  f32x4* part_o = reinterpret_cast<f32x4*>(smem);                    // [NT (keys)][NT (values)][64]
  f32x4* part_a = part_o + (OUT ? NT * NT * 64 : 0);                 // [NT][64]
  elt* vs = reinterpret_cast<elt*>(part_a + (OUT ? NT * 64 : 0));    // [NT][64][8] values as operands
  elt* zs = vs + NT * 512;                                           // [2][3 TC_RK][64][8] the decays' operands of this chunk and the next
  float* ssq = reinterpret_cast<float*>(zs + 2 * 3 * TC_RK * 512);   // [NT][16]
  const TimeMixRange rg = ranges[blockIdx.y];
  if (rg.slot < 0 || rg.slot >= a.n_seq || rg.tokens <= 0 || (!OUT && rg.add < 0)) return;   // uniform
  const int h = blockIdx.x, D = FULL ? 16 * NT : a.D, hd = h * D;
  const int w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, q16 = lane & 15, g = lane >> 4;
  const int d0 = 16 * w + 4 * g;                                     // this lane's four keys (and, of the outputs, values)
  const float LOG2E = 1.44269504088896340736f;
  f32x4 w0 = f32x4{0.f, 0.f, 0.f, 0.f}, u4 = w0, nw = w0;
#pragma unroll
  for (int e = 0; e < 4; ++e)
    if (FULL || d0 + e < D) {
      w0[e] = a.w0[hd + d0 + e] * LOG2E;
      u4[e] = a.u[hd + d0 + e];
      nw[e] = (float)a.norm[hd + d0 + e];
    }
  auto load4 = [&](const elt* p, uint32_t row) {                     // columns d0 .. d0 + 3 of a row, zero behind the head
    if constexpr (FULL) {
      return *reinterpret_cast<const u32x2*>(p + (row + (uint32_t)(hd + d0)));
    } else {
      eltx4 v = eltx4{0, 0, 0, 0};
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (d0 + e < D) v[e] = p[row + (uint32_t)(hd + d0 + e)];
      return __builtin_bit_cast(u32x2, v);
    }
  };
  const elt* w2p = a.w2 + (size_t)(hd + (FULL || 16 * w + q16 < D ? 16 * w + q16 : D - 1)) * rb * 32 + g * 8;
  eltx8 w2r[TC_RK];
#pragma unroll
  for (int i = 0; i < TC_RK; ++i) w2r[i] = ld8(w2p + (i < rb ? i : 0) * 32);
  // identity operands: slot (g, e) is column 4 g + e, of the hi half or of the lo half
  eltx8 idh, idl;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const elt one = (elt)(4 * g + e == q16 ? 1.f : 0.f);
    idh[e] = idl[4 + e] = one;
    idh[4 + e] = idl[e] = (elt)0.f;
  }

  // the state: S[n][r] = keys d0 + r, value 16 n + q16
  f32x4 S[NT], keep = f32x4{1.f, 1.f, 1.f, 1.f};                     // keep (OUT false): the range's decay
  const float* sp = rg.in >= 0 ? scratch + ((size_t)rg.in * a.H + h) * D * D : a.state + ((size_t)rg.slot * a.H + h) * D * D;
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    S[n] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (OUT && (rg.in >= 0 || rg.pos > 0)) {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (FULL || (d0 + r < D && 16 * n + q16 < D)) S[n][r] = sp[(d0 + r) * D + 16 * n + q16];
    }
  }

  const int steps = (rg.tokens + 15) / 16, tl = rg.tokens - 1;
  // a chunk's inputs, requested one chunk ahead (tokens behind the range repeat its last one; their keys and queries are cleared)
  u32x2 r_n = u32x2{0, 0}, k_n, v_n, g_n = r_n;
  const int nk = rb < TC_RK ? rb : TC_RK;
  auto row_of = [&](int c) { return (uint32_t)(rg.first + (c * 16 + q16 < tl ? c * 16 + q16 : tl)); };
  auto request = [&](int c) {
    const uint32_t t = row_of(c), row = t * (uint32_t)a.ld, zr = t * (uint32_t)(3 * 32 * rb) + g * 8;
    for (int f = w; f < 3 * nk; f += NT) {                           // uniform: fragment p nk + i, shared by the waves
      const int p = f / nk, i = f - p * nk;
      __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(zp + (zr + (uint32_t)((p * rb + i) * 32))),
                                       (__attribute__((address_space(3))) void*)(zs + ((c & 1) * 3 * TC_RK + f) * 512), 16, 0, 0);
    }
    k_n = load4(a.k, row);
    v_n = load4(a.v, row);
    if (OUT) {
      r_n = load4(a.r, row);
      g_n = load4(a.g, row);
    }
  };
  // a chunk's requests have landed (the wave's, then everybody's)
  auto landed = [&]() {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    lds_barrier();
  };
  request(0);
  landed();
  for (int c = 0; c < steps; ++c) {
    const bool live = c * 16 + q16 <= tl;
    const f32x4 g4 = floats(g_n);
    f32x4 r4 = floats(r_n), k4 = floats(k_n);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      r4[e] = live ? r4[e] : 0.f;
      k4[e] = live ? k4[e] : 0.f;
    }
    // values as operands: value 16 w + q16 of tokens 4 g .. + 3
    const f32x4 vt = mfma_16x16x32(operand(v_n[0], v_n[1], 0u, 0u), idh, f32x4{0.f, 0.f, 0.f, 0.f});
    const u32x2 v2 = __builtin_bit_cast(u32x2, __builtin_convertvector(vt, eltx4));
    const eltx8 vv = operand(v2[0], v2[1], v2[0], v2[1]);
    // logarithm (base 2) of the decays: lane (token q16; keys d0 ..)
    f32x4 lw = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < TC_RK; ++i)
      if (i < nk) {                                                  // uniform
#pragma unroll
        for (int p = 0; p < 3; ++p) lw = mfma_16x16x32(w2r[i], ld8(zs + ((c & 1) * 3 * TC_RK + p * nk + i) * 512 + lane * 8), lw);
      }
    for (int i = TC_RK; i < rb; ++i) {
      const eltx8 wi = ld8(w2p + i * 32);
      const uint32_t zr = row_of(c) * (uint32_t)(3 * 32 * rb) + g * 8;
#pragma unroll
      for (int p = 0; p < 3; ++p) lw = mfma_16x16x32(wi, ld8(zp + (zr + (uint32_t)((p * rb + i) * 32))), lw);
    }
    if (c + 1 < steps) request(c + 1);                               // uniform
    f32x4 Li, Lx, Lt;                                                // sums up to this token, without it, of the chunk
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      float x = live ? -LOG2E * __builtin_amdgcn_exp2f(fmaf(lw[e], LOG2E, w0[e])) : 0.f;
      x += row_shr<1>(x);
      x += row_shr<2>(x);
      x += row_shr<4>(x);
      x += row_shr<8>(x);
      Li[e] = x;
      Lx[e] = row_shr<1>(x);
      Lt[e] = row_lane<15>(x);
    }
    const f32x4 dec = exp2_4(Lt);
    // keys as the state takes them: three parts, all of fp32
    const f32x4 kf = k4 * exp2_4(Lt - Li);
    const HiLo kd(kf);
    const u32x2 ke = __builtin_bit_cast(u32x2, __builtin_convertvector(kf - floats(u32x2{kd.h[0], kd.h[1]}) - floats(u32x2{kd.l[0], kd.l[1]}), eltx4));
    st8(vs + (w * 64 + lane) * 8, vv);
    if constexpr (OUT) {
      // this wave's keys' part of A: A^T[s = 4 g + r][t = q16]
      const f32x4 ru = r4 * u4;
      float bs = fmaf(ru[0], k4[0], ru[1] * k4[1]) + fmaf(ru[2], k4[2], ru[3] * k4[3]);
      bs += __shfl_xor(bs, 16, WAVE);
      bs += __shfl_xor(bs, 32, WAVE);
      f32x4 A;
#pragma unroll
      for (int r = 0; r < 4; ++r) A[r] = 4 * g + r == q16 ? bs : 0.f;
      auto level = [&](auto HB, const f32x4& m) {                    // m: the sum up to the middle of the token's block of 2 h
        constexpr int hb = decltype(HB)::value;
        const bool up = q16 & hb;
        f32x4 x;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          x[e] = up ? r4[e] : k4[e];
          if (hb > 1) x[e] *= __builtin_amdgcn_exp2f(-fabsf((up ? Lx[e] : Li[e]) - m[e]));   // Lx <= m <= L on the two sides
        }
        const HiLo p(x);
        f32x4 G;
        if (hb > 1) {
          const eltx8 b = both(p);
          G = mfma_16x16x32(b, b, f32x4{0.f, 0.f, 0.f, 0.f});
          G = mfma_16x16x32(b, swapped(p), G);
        } else {                                                     // r and k themselves: elements
          G = mfma_16x16x32(operand(p.h[0], p.h[1], 0u, 0u), operand(p.h[0], p.h[1], 0u, 0u), f32x4{0.f, 0.f, 0.f, 0.f});
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int d = (4 * g + r) ^ q16;
          A[r] = up && d >= hb && d < 2 * hb ? G[r] : A[r];
        }
      };
      f32x4 m8, m4, m2;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        m8[e] = row_lane<7>(Li[e]);
        const float lo = row_lane<3>(Li[e]), hi = row_lane<11>(Li[e]);
        m4[e] = q16 & 8 ? hi : lo;
        m2[e] = quad_lane1(Li[e]);
      }
      level(std::integral_constant<int, 8>(), m8);
      level(std::integral_constant<int, 4>(), m4);
      level(std::integral_constant<int, 2>(), m2);
      level(std::integral_constant<int, 1>(), Li);
      part_a[w * 64 + lane] = A;
      // ... and of what comes out of the state: o^T[value 16 n + 4 g + r][t = q16]
      const HiLo R(r4 * exp2_4(Lx));
      const eltx8 ra = both(R), rs = swapped(R);
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        const eltx8 s8 = both(HiLo(S[n]));
        const f32x4 o = mfma_16x16x32(s8, ra, f32x4{0.f, 0.f, 0.f, 0.f});
        part_o[(w * NT + n) * 64 + lane] = mfma_16x16x32(s8, rs, o);
      }
    }
    lds_barrier();
    // the state takes the chunk
    {
      const eltx8 kb = both(kd);
      const f32x4 th = mfma_16x16x32(kb, idh, f32x4{0.f, 0.f, 0.f, 0.f}), tlo = mfma_16x16x32(kb, idl, f32x4{0.f, 0.f, 0.f, 0.f});   // [s = 4 g + r][key 16 w + q16]
      const u32x2 uh = __builtin_bit_cast(u32x2, __builtin_convertvector(th, eltx4)), ul = __builtin_bit_cast(u32x2, __builtin_convertvector(tlo, eltx4));
      const f32x4 te = mfma_16x16x32(operand(ke[0], ke[1], 0u, 0u), idh, f32x4{0.f, 0.f, 0.f, 0.f});
      const u32x2 ue = __builtin_bit_cast(u32x2, __builtin_convertvector(te, eltx4));
      const eltx8 kt = operand(uh[0], uh[1], ul[0], ul[1]), kr = operand(ue[0], ue[1], 0u, 0u);
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        const eltx8 v = ld8(vs + (n * 64 + lane) * 8);
        S[n] = mfma_16x16x32(kr, v, mfma_16x16x32(kt, v, S[n] * dec));
      }
      if (!OUT) keep *= dec;
    }
    if constexpr (OUT) {
      f32x4 A = part_a[lane], o = part_o[w * 64 + lane];
#pragma unroll
      for (int i = 1; i < NT; ++i) {
        A += part_a[i * 64 + lane];
        o += part_o[(i * NT + w) * 64 + lane];
      }
      o = mfma_16x16x32(vv, both(HiLo(A)), o);                // o^T[value d0 + r][t = q16]
      float ss = fmaf(o[0], o[0], o[1] * o[1]) + fmaf(o[2], o[2], o[3] * o[3]);
      ss += __shfl_xor(ss, 16, WAVE);
      ss += __shfl_xor(ss, 32, WAVE);
      if (g == 0) ssq[w * 16 + q16] = ss;
      landed();
      float tot = ssq[q16];
#pragma unroll
      for (int i = 1; i < NT; ++i) tot += ssq[i * 16 + q16];
      const float inv = __builtin_amdgcn_rsqf(fmaf(tot, 1.f / (float)D, a.eps));
      f32x4 y;
#pragma unroll
      for (int e = 0; e < 4; ++e) y[e] = o[e] * inv * nw[e] * (g4[e] * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-LOG2E * g4[e])));
      const eltx4 y4 = __builtin_convertvector(y, eltx4);
      if (live) {
        const int t = rg.first + c * 16 + q16;
        if constexpr (FULL) {
          *reinterpret_cast<eltx4*>(a.y + (a.frag_tt ? frag_offset(t, hd + d0, a.frag_tt) : (size_t)t * a.ld_y + hd + d0)) = y4;
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (d0 + e < D) a.y[a.frag_tt ? frag_offset(t, hd + d0 + e, a.frag_tt) : (size_t)t * a.ld_y + hd + d0 + e] = y4[e];
        }
      }
    } else {
      landed();
    }
  }
  float* so = OUT ? a.state + ((size_t)rg.slot * a.H + h) * D * D : scratch + ((size_t)rg.add * a.H + h) * D * D;
  if (!OUT || rg.last) {
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (FULL || (d0 + r < D && 16 * n + q16 < D)) so[(d0 + r) * D + 16 * n + q16] = S[n][r];
  }
  if (!OUT && q16 == 0) {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (FULL || d0 + e < D) decay[((size_t)rg.add * a.H + h) * D + d0 + e] = keep[e];
  }
}

// scratch states first .. first + count - 1 of a sequence: what its ranges add (all but the last) becomes the state ahead of each
struct TimeMixSeq {         // 4 int32
  int slot, pos, first, count;
};
__global__ __launch_bounds__(256) void time_mix_range_kernel(const float* __restrict__ state, float* __restrict__ scratch, const float* __restrict__ decay,
                                                             const TimeMixSeq* __restrict__ seqs, int n_seq, int H, int D) {
  const TimeMixSeq q = seqs[blockIdx.z];
  const int h = blockIdx.y, i = blockIdx.x * 256 + threadIdx.x;
  if (q.slot < 0 || q.slot >= n_seq || i >= D * D) return;
  float s = q.pos > 0 ? state[((size_t)q.slot * H + h) * D * D + i] : 0.f;
  const int row = i / D;
  constexpr int U = 8;                                               // ranges requested together
  for (int c0 = 0; c0 < q.count; c0 += U) {
    float add[U], w[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const bool in = c0 + u + 1 < q.count;
      const size_t at = (size_t)(q.first + (in ? c0 + u : 0)) * H + h;
      add[u] = in ? scratch[at * D * D + i] : 0.f;
      w[u] = in ? decay[at * D + row] : 0.f;
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (c0 + u < q.count) scratch[((size_t)(q.first + c0 + u) * H + h) * D * D + i] = s;
      s = fmaf(w[u], s, add[u]);
    }
  }
}
#endif

// the columns behind the heads, read by the matrix cores as zeros
__global__ __launch_bounds__(64) void time_mix_pad_kernel(elt* __restrict__ y, int frag_tt, int ld_y, int c0) {
  const int t = blockIdx.x, c = c0 + threadIdx.x;
  if (c < ld_y) y[frag_tt ? frag_offset(t, c, frag_tt) : (size_t)t * ld_y + c] = (elt)0.f;
}

}  // namespace

extern "C" int mlora_time_mix(void* y, int y_layout, int ld_y, const void* r, const void* k, const void* v, const void* g, int ld, const float* z,
                              int n_z, int ld_z, int R, const void* w2, int ld_w2, const float* w0, const float* u, const void* norm, float eps, float* state,
                              int n_seq, const int32_t* segs, int n_segs, const int32_t* tok_seq, const int32_t* tok_pos, int T, int H, int D,
                              void* stream) {
  MLORA_CHECK(y && r && k && v && g && z && w2 && w0 && u && norm && state && (segs || (tok_seq && tok_pos)), MLORA_ERR_INVALID, "time_mix: null pointer");
  MLORA_CHECK(T >= 0 && H > 0 && D > 0 && D <= 256 && n_z >= 1 && R > 0 && R <= TM_MAX_R && ld >= H * D && ld_z >= R && ld_w2 >= R && ld_w2 % 8 == 0 && ld_w2 <= TM_MAX_R && ld_y >= H * D &&
                  ld_y < H * D + 64 && n_seq > 0 && n_segs >= 0 && n_segs <= 65535 && (segs || n_segs == T),
              MLORA_ERR_UNSUPPORTED, "time_mix: need heads of at most 256 channels and a decay rank of at most %d (T=%d H=%d D=%d R=%d)", TM_MAX_R, T, H, D, R);
  MLORA_CHECK(y_layout == MLORA_ROWMAJOR || (ld_y % 32 == 0 && sizeof(elt) == 2), MLORA_ERR_UNSUPPORTED, "time_mix: fragment order needs whole blocks of 32");
  if (T == 0 || n_segs == 0) return MLORA_OK;
  TimeMix a;
  a.y = (elt*)y; a.frag_tt = y_layout == MLORA_FRAG ? mlora_frag_tiles(T) : 0; a.ld_y = ld_y;
  a.r = (const elt*)r; a.k = (const elt*)k; a.v = (const elt*)v; a.g = (const elt*)g; a.ld = ld; a.z = z; a.n_z = n_z; a.ld_z = ld_z; a.R = R;
  a.w2 = (const elt*)w2; a.ld_w2 = ld_w2; a.w0 = w0; a.u = u; a.norm = (const elt*)norm; a.eps = eps; a.state = state; a.n_seq = n_seq;
  a.H = H; a.D = D; a.T = T; a.segs = (const int4*)segs; a.tok_seq = tok_seq; a.tok_pos = tok_pos;
  hipStream_t s = (hipStream_t)stream;
  const dim3 grid(H, n_segs);
  if (!segs && D <= 128) {                     // a decode step
    if (D <= 32) hipLaunchKernelGGL(time_mix_step_kernel<32>, grid, dim3(TS_THREADS), 0, s, a);
    else if (D <= 64) hipLaunchKernelGGL(time_mix_step_kernel<64>, grid, dim3(TS_THREADS), 0, s, a);
    else hipLaunchKernelGGL(time_mix_step_kernel<128>, grid, dim3(TS_THREADS), 0, s, a);
  } else if (D <= 64) hipLaunchKernelGGL((time_mix_scan_kernel<8, 64, 8, 8>), grid, dim3(512), 0, s, a);
  else if (D <= 128) hipLaunchKernelGGL((time_mix_scan_kernel<16, 128, 8, 4>), grid, dim3(1024), 0, s, a);
  else hipLaunchKernelGGL((time_mix_scan_kernel<64, 256, 4, 4>), grid, dim3(1024), 0, s, a);
  if (ld_y > H * D) hipLaunchKernelGGL(time_mix_pad_kernel, dim3(T), dim3(64), 0, s, a.y, a.frag_tt, ld_y, H * D);
  return mlora_launch_status("time_mix");
}

#ifndef MLORA_ELT_F32
template <int NT, bool FULL, bool OUT>
static int launch_time_mix_chunk(const TimeMix& a, const void* zp, int rb, const int32_t* ranges, int n_ranges, float* scratch, float* decay, hipStream_t s) {
  constexpr size_t lds = (OUT ? (size_t)(NT * NT + NT) * 1024 : 0) + (size_t)(NT + 2 * 3 * TC_RK) * 1024 + NT * 64;
  static const hipError_t configured =               // the attribute is per kernel, set once per process, by one thread
      hipFuncSetAttribute((const void*)time_mix_chunk_kernel<NT, FULL, OUT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  if (configured != hipSuccess) return mlora_set_error(MLORA_ERR_LAUNCH, "time_mix_prompt: cannot reserve %zu bytes of LDS", lds);
  hipLaunchKernelGGL((time_mix_chunk_kernel<NT, FULL, OUT>), dim3(a.H, n_ranges), dim3(NT * WAVE), lds, s, a, (const elt*)zp, rb,
                     (const TimeMixRange*)ranges, scratch, decay);
  return MLORA_OK;
}

extern "C" int mlora_time_mix_prompt_served(int D) { return D > 0 && D <= 128; }

extern "C" int mlora_time_mix_prompt(void* y, int y_layout, int ld_y, const void* r, const void* k, const void* v, const void* g, int ld, const void* zp,
                                     int ld_zp, const void* w2, const float* w0, const float* u, const void* norm, float eps, float* state, int n_seq,
                                     const int32_t* ranges, int n_ranges, const int32_t* seqs, int n_seqs, float* scratch, size_t scratch_floats,
                                     int n_states, int T, int H, int D, void* stream) {
  MLORA_CHECK(y && r && k && v && g && zp && w2 && w0 && u && norm && state && ranges && (n_seqs == 0 || (seqs && scratch)), MLORA_ERR_INVALID,
              "time_mix_prompt: null pointer");
  MLORA_CHECK(T >= 0 && H > 0 && H <= 65535 && mlora_time_mix_prompt_served(D) && ld >= H * D && ld % 4 == 0 && ld_zp > 0 && ld_zp % 32 == 0 && ld_y >= H * D &&
                  ld_y < H * D + 64 && n_seq > 0 && n_ranges >= 0 && n_ranges <= 65535 && n_seqs >= 0 && n_seqs <= 65535 && n_states >= 0 &&
                  (((uintptr_t)zp | (uintptr_t)w2) & 15) == 0,
              MLORA_ERR_UNSUPPORTED, "time_mix_prompt: need heads of at most 128 channels (T=%d H=%d D=%d)", T, H, D);
  MLORA_CHECK((long)T * ld < (1L << 31) && (long)T * 3 * ld_zp < (1L << 31) && (((uintptr_t)r | (uintptr_t)k | (uintptr_t)v | (uintptr_t)g) & 7) == 0,
              MLORA_ERR_UNSUPPORTED, "time_mix_prompt: T=%d is too many tokens for rows of %d, or unaligned operands", T, ld);
  MLORA_CHECK(y_layout == MLORA_ROWMAJOR || ld_y % 32 == 0, MLORA_ERR_UNSUPPORTED, "time_mix_prompt: fragment order needs whole blocks of 32");
  MLORA_CHECK(n_seqs == 0 || scratch_floats >= (size_t)n_states * H * D * (D + 1), MLORA_ERR_WORKSPACE, "time_mix_prompt: scratch too small");
  if (T == 0 || n_ranges == 0) return MLORA_OK;
  TimeMix a = {};
  a.y = (elt*)y; a.frag_tt = y_layout == MLORA_FRAG ? mlora_frag_tiles(T) : 0; a.ld_y = ld_y;
  a.r = (const elt*)r; a.k = (const elt*)k; a.v = (const elt*)v; a.g = (const elt*)g; a.ld = ld; a.w0 = w0; a.u = u; a.norm = (const elt*)norm;
  a.eps = eps; a.state = state; a.n_seq = n_seq; a.H = H; a.D = D; a.T = T; a.w2 = (const elt*)w2;
  float* decay = scratch + (size_t)n_states * H * D * D;
  const int rb = ld_zp / 32;
  hipStream_t s = (hipStream_t)stream;
  int e = MLORA_OK;
  auto launch = [&](auto OUT) {
    constexpr bool out = decltype(OUT)::value;
    if (D == 64) return launch_time_mix_chunk<4, true, out>(a, zp, rb, ranges, n_ranges, scratch, decay, s);
    if (D == 128) return launch_time_mix_chunk<8, true, out>(a, zp, rb, ranges, n_ranges, scratch, decay, s);
    if (D <= 32) return launch_time_mix_chunk<2, false, out>(a, zp, rb, ranges, n_ranges, scratch, decay, s);
    if (D <= 64) return launch_time_mix_chunk<4, false, out>(a, zp, rb, ranges, n_ranges, scratch, decay, s);
    return launch_time_mix_chunk<8, false, out>(a, zp, rb, ranges, n_ranges, scratch, decay, s);
  };
  if (n_seqs > 0) {
    e = launch(std::false_type());
    if (e) return e;
    hipLaunchKernelGGL(time_mix_range_kernel, dim3(ceil_div(D * D, 256), H, n_seqs), dim3(256), 0, s, state, scratch, decay, (const TimeMixSeq*)seqs, n_seq,
                       H, D);
  }
  e = launch(std::true_type());
  if (e) return e;
  if (ld_y > H * D) hipLaunchKernelGGL(time_mix_pad_kernel, dim3(T), dim3(64), 0, s, a.y, a.frag_tt, ld_y, H * D);
  return mlora_launch_status("time_mix_prompt");
}
#endif
