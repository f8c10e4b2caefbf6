// Time mixing with a matrix state per head and a decay per key channel (a linear recurrence):
//     o_t = (S + diag(u) k_t v_t^T)^T r_t        S <- diag(w_t) S + k_t v_t^T
//     w_t = exp(-exp(W2 tanh(z_t) + w0))         z_t: the decay's low-rank projection of the token
//     y_t = o_t / rms(o_t) * norm * silu(g_t)    rms over the head
// r, k, v, g [T, ld] in elements (columns head * D + channel), z [T, ld_z] fp32; everything behind the projections is fp32.
// The state [n_seq, H, D (key), D (value)] fp32 belongs to a sequence's slot; a sequence whose first token of the pass has
// position 0 starts from zero, whatever the slot holds.  Compiled for every element type.
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
  const float* z;           // [T, ld_z], R columns count
  int ld_z, R;
  const elt* w2t;           // [R, ld_w2]: W2 transposed
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
    for (int i = threadIdx.x; i < n * a.R; i += NT) {
      const int t = i / a.R, j = i - t * a.R;
      zs[t][j] = tanhf(a.z[(size_t)(tb + t) * a.ld_z + j]);
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
        for (int j = 0; j < a.R; ++j) s = fmaf(zs[t][j], (float)a.w2t[(size_t)j * a.ld_w2 + hd + d], s);
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

// the columns behind the heads, read by the matrix cores as zeros
__global__ __launch_bounds__(64) void time_mix_pad_kernel(elt* __restrict__ y, int frag_tt, int ld_y, int c0) {
  const int t = blockIdx.x, c = c0 + threadIdx.x;
  if (c < ld_y) y[frag_tt ? frag_offset(t, c, frag_tt) : (size_t)t * ld_y + c] = (elt)0.f;
}

}  // namespace

extern "C" int mlora_time_mix(void* y, int y_layout, int ld_y, const void* r, const void* k, const void* v, const void* g, int ld, const float* z,
                              int ld_z, int R, const void* w2t, int ld_w2, const float* w0, const float* u, const void* norm, float eps, float* state,
                              int n_seq, const int32_t* segs, int n_segs, const int32_t* tok_seq, const int32_t* tok_pos, int T, int H, int D,
                              void* stream) {
  MLORA_CHECK(y && r && k && v && g && z && w2t && w0 && u && norm && state && (segs || (tok_seq && tok_pos)), MLORA_ERR_INVALID, "time_mix: null pointer");
  MLORA_CHECK(T >= 0 && H > 0 && D > 0 && D <= 256 && R > 0 && R <= TM_MAX_R && ld >= H * D && ld_z >= R && ld_w2 >= H * D && ld_y >= H * D &&
                  ld_y < H * D + 64 && n_seq > 0 && n_segs >= 0 && n_segs <= 65535 && (segs || n_segs == T),
              MLORA_ERR_UNSUPPORTED, "time_mix: need heads of at most 256 channels and a decay rank of at most %d (T=%d H=%d D=%d R=%d)", TM_MAX_R, T, H, D, R);
  MLORA_CHECK(y_layout == MLORA_ROWMAJOR || (ld_y % 32 == 0 && sizeof(elt) == 2), MLORA_ERR_UNSUPPORTED, "time_mix: fragment order needs whole blocks of 32");
  if (T == 0 || n_segs == 0) return MLORA_OK;
  TimeMix a;
  a.y = (elt*)y; a.frag_tt = y_layout == MLORA_FRAG ? mlora_frag_tiles(T) : 0; a.ld_y = ld_y;
  a.r = (const elt*)r; a.k = (const elt*)k; a.v = (const elt*)v; a.g = (const elt*)g; a.ld = ld; a.z = z; a.ld_z = ld_z; a.R = R;
  a.w2t = (const elt*)w2t; a.ld_w2 = ld_w2; a.w0 = w0; a.u = u; a.norm = (const elt*)norm; a.eps = eps; a.state = state; a.n_seq = n_seq;
  a.H = H; a.D = D; a.T = T; a.segs = (const int4*)segs; a.tok_seq = tok_seq; a.tok_pos = tok_pos;
  hipStream_t s = (hipStream_t)stream;
  const dim3 grid(H, n_segs);
  if (D <= 64) hipLaunchKernelGGL((time_mix_scan_kernel<8, 64, 8, 8>), grid, dim3(512), 0, s, a);
  else if (D <= 128) hipLaunchKernelGGL((time_mix_scan_kernel<16, 128, 8, 4>), grid, dim3(1024), 0, s, a);
  else hipLaunchKernelGGL((time_mix_scan_kernel<64, 256, 4, 4>), grid, dim3(1024), 0, s, a);
  if (ld_y > H * D) hipLaunchKernelGGL(time_mix_pad_kernel, dim3(T), dim3(64), 0, s, a.y, a.frag_tt, ld_y, H * D);
  return mlora_launch_status("time_mix");
}
