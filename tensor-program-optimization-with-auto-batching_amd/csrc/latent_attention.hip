// Latent attention: keys and values of all heads are linear images of one cached vector per token - the normed latent c
// (kv_rank) - beside one rotated key part shared by the heads (rot_dim).  The score of head h is
//     (W_uk[h]^T q_h) . c  +  q_rot_h . k_rot
// and its output W_uv[h] . sum_j p_j c_j, so the attention kernels work on the latents alone: queries are lifted into the
// latent space first (mlora_head_linear over W_uk), the context vectors leave it afterwards (over W_uv).
//
// Cache of a layer: [n_pages, NB, 4, 16, 8] elements, NB = RB + rotation blocks; element (token, d) of a page at
// ((d/32 * 4 + (d%32)/8) * 16 + token) * 8 + d%8 - the page layout of the K cache of attention.hip with one head.  The
// latent takes the first RB = ceil(kv_rank / 32) blocks, the rotated part the following ones, padding is zero.
// There is no second copy for the values: the matrix cores transpose a page's fragments by a product with the identity.
// Query rows: [T, H, NB * 32] in the same order.
#include "common.h"

namespace {

constexpr int PAGE = MLORA_PAGE_SIZE;

__device__ __forceinline__ size_t latent_offset(int page, int NB, int token, int d) {
  return (size_t)page * NB * 512 + ((((d >> 5) * 4 + ((d >> 3) & 3)) * PAGE + token) * 8 + (d & 7));
}

struct LatentPrep {
  const elt* qkv;           // [T, ld]: projections of a token, not yet scaled by `gain`
  int ld, off_rot, off_c, off_kr;   // columns of the heads' rotated query parts [H, rot], of the latent and of the key part
  float gain, eps;
  const elt* c_norm;        // [R] weight of the latent's norm; nullptr: the layer reads another layer's cache
  elt* cache;
  const int32_t* block_table;
  int max_blocks, n_pages, n_seq;
  const int32_t* tok_seq;
  const int32_t* tok_pos;
  const float* cos;         // [max_pos, rot / 2]
  const float* sin;
  int max_pos, H, R, rot, RB, NB;
  elt* q;                   // [T, H, NB * 32]: the rotated part is written here
};

// One workgroup per token: rotates the heads' query parts into the query rows, norms the latent, rotates the shared key
// part and stores both in the token's page slot.  Neighbouring elements (2 i, 2 i + 1) turn by the table's angle i.
__global__ __launch_bounds__(256) void latent_prep_kernel(LatentPrep a) {
  __shared__ float red[4];
  const int t = blockIdx.x;
  const int seq = a.tok_seq[t], pos = a.tok_pos[t];
  if (seq < 0 || seq >= a.n_seq || pos < 0 || pos >= a.max_pos || pos / PAGE >= a.max_blocks) return;   // uniform
  const elt* row = a.qkv + (size_t)t * a.ld;
  const int half = a.rot / 2, qd = a.NB * 32, rp = (a.NB - a.RB) * 32;
  const float* cp = a.cos + (size_t)pos * half;
  const float* sp = a.sin + (size_t)pos * half;
  elt* q = a.q + (size_t)t * a.H * qd + a.RB * 32;
  for (int i = threadIdx.x; i < a.H * (rp / 2); i += 256) {
    const int h = i / (rp / 2), k = i - h * (rp / 2);
    float u = 0.f, v = 0.f;
    if (k < half) {
      const float x1 = (float)row[a.off_rot + h * a.rot + 2 * k] * a.gain, x2 = (float)row[a.off_rot + h * a.rot + 2 * k + 1] * a.gain;
      u = x1 * cp[k] - x2 * sp[k];
      v = x2 * cp[k] + x1 * sp[k];
    }
    *reinterpret_cast<eltx2*>(q + (size_t)h * qd + 2 * k) = eltx2{(elt)u, (elt)v};
  }
  if (!a.c_norm) return;
  const int page = a.block_table[(size_t)seq * a.max_blocks + pos / PAGE];
  float ss = 0.f;
  for (int d = threadIdx.x; d < a.R; d += 256) {
    const float c = (float)row[a.off_c + d] * a.gain;
    ss = fmaf(c, c, ss);
  }
  ss = wave_sum(ss);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
  __syncthreads();
  const float inv = a.gain / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.R + a.eps);
  if (page < 0 || page >= a.n_pages) return;
  for (int d = threadIdx.x; d < a.R; d += 256)
    a.cache[latent_offset(page, a.NB, pos % PAGE, d)] = (elt)((float)row[a.off_c + d] * inv * (float)a.c_norm[d]);
  for (int k = threadIdx.x; k < half; k += 256) {
    const float x1 = (float)row[a.off_kr + 2 * k] * a.gain, x2 = (float)row[a.off_kr + 2 * k + 1] * a.gain;
    *reinterpret_cast<eltx2*>(a.cache + latent_offset(page, a.NB, pos % PAGE, a.RB * 32 + 2 * k)) =
        eltx2{(elt)(x1 * cp[k] - x2 * sp[k]), (elt)(x2 * cp[k] + x1 * sp[k])};
  }
}

struct LatentAttn {
  elt* out;                 // [T, H, RB * 32] sum_j p_j c_j
  float* part_o;            // splits > 1: [splits, T, H, RB * 32] unnormalised sums ...
  float* part_ml;           // ... and [splits, T, H, 2] their maximum and denominator
  const elt* q;             // [T, H, NB * 32]
  const elt* cache;
  const int32_t* block_table;
  int max_blocks, n_pages, n_seq;
  const int32_t* tok_seq;
  const int32_t* tok_pos;
  const float* sink;        // [H]
  float scale;
  int T, H, RB, NB, splits, n_inner, chunks;
};

// the context a token sees: every position up to its own
__device__ __forceinline__ int latent_ctx(const LatentAttn& a, int t, int& seq) {
  seq = a.tok_seq[t];
  int ctx = a.tok_pos[t] + 1;
  if (seq < 0 || seq >= a.n_seq || ctx < 0) ctx = 0;
  if (seq < 0 || seq >= a.n_seq) seq = 0;
  return ctx < a.max_blocks * PAGE ? ctx : a.max_blocks * PAGE;
}

#ifndef MLORA_ELT_F32
// A workgroup takes one token, 16 heads (the columns of the matrix-core tiles), a share of the context (split) and up to
// NRB blocks of the latent as output (chunk; all of it up to NRB blocks).  A wave takes every NW-th page:
//   S^T = K . Q^T        the page's fragments as they lie in the cache, queries from LDS
//   page^T               two products with halves of the identity per 32 dims: exact
//   O^T += page^T . P^T  P as hi + lo halves in the two halves of the k-slots, the page's values repeated in both
// The waves' states (m, l, O) meet in LDS, 64 dims at a time.
template <int NRB, int NW>
__global__ __launch_bounds__(NW * WAVE, 2) void latent_attn_kernel(LatentAttn a) {
  extern __shared__ __align__(16) char smem_raw[];
  elt* qs = reinterpret_cast<elt*>(smem_raw);                        // [NB][64][8] query fragments
  float* sacc = reinterpret_cast<float*>(qs + a.NB * 512);           // [NW][16][68]
  __shared__ float sm[NW][16], sl[NW][16];
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int col = lane & 15, g = lane >> 4;
  // the workgroups that walk the same pages (inner index: head groups and chunks) run on one XCD
  const int x8 = blockIdx.x & 7, rest = blockIdx.x >> 3;
  const int inner = rest % a.n_inner, outer = (rest / a.n_inner) * 8 + x8;
  if (outer >= a.T * a.splits) return;                               // uniform
  const int t = outer / a.splits, split = outer - t * a.splits;
  const int hg = inner / a.chunks, b0 = (inner - hg * a.chunks) * NRB;
  int seq;
  const int ctx = latent_ctx(a, t, seq);
  const int npages = (ctx + PAGE - 1) / PAGE;
  const int per = (npages + a.splits - 1) / a.splits;
  const int p0 = split * per, p1 = p0 + per < npages ? p0 + per : npages;
  const int32_t* __restrict__ bt = a.block_table + (size_t)seq * a.max_blocks;
  const int qd = a.NB * 32;

  for (int i = threadIdx.x; i < a.NB * 64; i += NW * WAVE) {
    const int kb = i >> 6, l = i & 63, h = hg * 16 + (l & 15);
    eltx8 v = eltx8{0, 0, 0, 0, 0, 0, 0, 0};
    if (h < a.H) v = ld8(a.q + ((size_t)t * a.H + h) * qd + kb * 32 + (l >> 4) * 8);
    st8(qs + i * 8, v);
  }
  // the identity's columns 0..15 and 16..31 as the B operand: lane (column col, k-group g) holds k = 8 g .. 8 g + 7
  eltx8 id0, id1;
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    id0[e] = (elt)(g * 8 + e == col ? 1.f : 0.f);
    id1[e] = (elt)(g * 8 + e == col + 16 ? 1.f : 0.f);
  }
  __syncthreads();

  float m = -INFINITY, l = 0.f;
  f32x4 O[2 * NRB];
#pragma unroll
  for (int db = 0; db < 2 * NRB; ++db) O[db] = f32x4{0.f, 0.f, 0.f, 0.f};

  for (int pg = p0 + wave; pg < p1; pg += NW) {
    const int page = bt[pg];
    if (page < 0 || page >= a.n_pages) continue;                     // wave-uniform
    const elt* kp = a.cache + (size_t)page * a.NB * 512 + lane * 8;
    eltx8 kf[NRB];
#pragma unroll
    for (int b = 0; b < NRB; ++b) {
      const int kb = b0 + b < a.RB ? b0 + b : a.RB - 1;
      kf[b] = ld8(kp + kb * 512);
    }
    f32x4 st = f32x4{0.f, 0.f, 0.f, 0.f};                            // st[r] = S[token 4 g + r][head col]
    for (int kb = a.RB; kb < a.NB; ++kb) st = mfma_16x16x32(ld8(kp + kb * 512), ld8(qs + (kb * 64 + lane) * 8), st);
    if (a.chunks > 1)                                                // the latent's blocks outside this chunk
      for (int kb = 0; kb < a.RB; ++kb)
        if (kb < b0 || kb >= b0 + NRB) st = mfma_16x16x32(ld8(kp + kb * 512), ld8(qs + (kb * 64 + lane) * 8), st);
#pragma unroll
    for (int b = 0; b < NRB; ++b)
      if (b0 + b < a.RB) st = mfma_16x16x32(kf[b], ld8(qs + ((b0 + b) * 64 + lane) * 8), st);   // uniform

    float pm = -INFINITY;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      st[r] = pg * PAGE + 4 * g + r >= ctx ? -INFINITY : st[r] * a.scale;
      pm = fmaxf(pm, st[r]);
    }
    pm = fmaxf(pm, __shfl_xor(pm, 16, WAVE));
    pm = fmaxf(pm, __shfl_xor(pm, 32, WAVE));
    const float m_new = fmaxf(m, pm);                                // finite: the first token of a visited page is < ctx
    const float alpha = __expf(m - m_new);
    eltx8 pa;
    float ps = 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float p = __expf(st[r] - m_new);
      ps += p;
      const elt hi = (elt)p;
      pa[r] = hi;
      pa[4 + r] = (elt)(p - (float)hi);
    }
    l = l * alpha + ps;                                              // the lane's share of its column's sum
    m = m_new;
#pragma unroll
    for (int b = 0; b < NRB; ++b) {
      if (b0 + b < a.RB) {                                           // uniform
        const f32x4 t0 = mfma_16x16x32(kf[b], id0, f32x4{0.f, 0.f, 0.f, 0.f}), t1 = mfma_16x16x32(kf[b], id1, f32x4{0.f, 0.f, 0.f, 0.f});
        const eltx8 v0 = eltx8{(elt)t0[0], (elt)t0[1], (elt)t0[2], (elt)t0[3], (elt)t0[0], (elt)t0[1], (elt)t0[2], (elt)t0[3]};
        const eltx8 v1 = eltx8{(elt)t1[0], (elt)t1[1], (elt)t1[2], (elt)t1[3], (elt)t1[0], (elt)t1[1], (elt)t1[2], (elt)t1[3]};
        O[2 * b] *= alpha;
        O[2 * b + 1] *= alpha;
        O[2 * b] = mfma_16x16x32(v0, pa, O[2 * b]);                  // O^T[dim 32 b + 4 g + r][head col]
        O[2 * b + 1] = mfma_16x16x32(v1, pa, O[2 * b + 1]);
      }
    }
  }
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  if (g == 0) {
    sm[wave][col] = m;
    sl[wave][col] = l;
  }
#pragma unroll
  for (int c = 0; c < NRB; c += 2) {                                 // 64 dims
    if (b0 + c < a.RB) {                                             // uniform
      __syncthreads();
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (2 * c + u < 2 * NRB) *reinterpret_cast<f32x4*>(sacc + (wave * 16 + col) * 68 + u * 16 + 4 * g) = O[(2 * c + u) % (2 * NRB)];
      __syncthreads();
      for (int e = threadIdx.x; e < 16 * 64; e += NW * WAVE) {
        const int hc = e >> 6, dd = e & 63, h = hg * 16 + hc, d = (b0 + c) * 32 + dd;
        if (h >= a.H || d >= a.RB * 32 || d >= (b0 + NRB) * 32) continue;
        float M = sm[0][hc];
#pragma unroll
        for (int w = 1; w < NW; ++w) M = fmaxf(M, sm[w][hc]);
        const float sk = a.sink ? a.sink[h] : -INFINITY;
        if (a.splits == 1) M = fmaxf(M, sk);
        float L = 0.f, o = 0.f;
#pragma unroll
        for (int w = 0; w < NW; ++w) {
          const float f = sm[w][hc] == -INFINITY ? 0.f : __expf(sm[w][hc] - M);
          L += sl[w][hc] * f;
          o += sacc[(w * 16 + hc) * 68 + dd] * f;
        }
        if (a.splits == 1) {
          if (sk != -INFINITY) L += __expf(sk - M);
          a.out[((size_t)t * a.H + h) * (a.RB * 32) + d] = (elt)(L > 0.f ? o / L : 0.f);
        } else {
          const size_t r = ((size_t)split * a.T + t) * a.H + h;
          a.part_o[r * (a.RB * 32) + d] = o;
          if (d == 0) {
            a.part_ml[2 * r] = M;
            a.part_ml[2 * r + 1] = L;
          }
        }
      }
    }
  }
}

// adds the splits of a (token, head) and the sink's share of the denominator
__global__ __launch_bounds__(128) void latent_merge_kernel(LatentAttn a) {
  const int th = blockIdx.x, h = th % a.H, rd = a.RB * 32;
  const size_t n = (size_t)a.T * a.H;
  const float sk = a.sink ? a.sink[h] : -INFINITY;
  float M = sk;
  for (int s = 0; s < a.splits; ++s) M = fmaxf(M, a.part_ml[2 * (s * n + th)]);
  float L = sk != -INFINITY ? __expf(sk - M) : 0.f;
  for (int s = 0; s < a.splits; ++s) {
    const float m = a.part_ml[2 * (s * n + th)];
    if (m != -INFINITY) L += a.part_ml[2 * (s * n + th) + 1] * __expf(m - M);
  }
  const float inv = L > 0.f ? 1.f / L : 0.f;
  for (int d = threadIdx.x * 4; d < rd; d += 512) {
    f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < a.splits; ++s) {
      const float m = a.part_ml[2 * (s * n + th)];
      if (m != -INFINITY) o += *reinterpret_cast<const f32x4*>(a.part_o + (s * n + th) * rd + d) * __expf(m - M);
    }
    *reinterpret_cast<eltx4*>(a.out + (size_t)th * rd + d) = eltx4{(elt)(o[0] * inv), (elt)(o[1] * inv), (elt)(o[2] * inv), (elt)(o[3] * inv)};
  }
}

// y[t, h] = alpha * W[h] . x[t, h] per head: W[h] packed [N, K], N % 16 == 0.  A wave owns 16 NI rows x 16 TJ tokens.
template <int NI, int TJ>
__global__ __launch_bounds__(256) void head_linear_kernel(elt* __restrict__ y, long ldy, long hy, int frag_tt, const elt* __restrict__ x, long ldx,
                                                          long hx, const elt* __restrict__ Wp, int T, int K, int N, float alpha) {
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int h = blockIdx.z, t0 = blockIdx.y * 16 * TJ;
  const int KB = K / 32, tiles = N / 16, nt0 = (blockIdx.x * 4 + wave) * NI;
  if (nt0 >= tiles) return;
  const int r16 = lane & 15, g = lane >> 4;
  const elt* wp[NI];
  const elt* xp[TJ];
#pragma unroll
  for (int i = 0; i < NI; ++i) wp[i] = Wp + ((size_t)h * tiles + (nt0 + i < tiles ? nt0 + i : tiles - 1)) * KB * 512 + lane * 8;
#pragma unroll
  for (int j = 0; j < TJ; ++j) {
    const int t = t0 + j * 16 + r16;
    xp[j] = x + (t < T ? t : T - 1) * ldx + h * hx + g * 8;
  }
  f32x4 acc[NI][TJ];
#pragma unroll
  for (int i = 0; i < NI; ++i)
#pragma unroll
    for (int j = 0; j < TJ; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int ks = 0; ks < KB; ++ks) {
    eltx8 w[NI], b[TJ];
#pragma unroll
    for (int i = 0; i < NI; ++i) w[i] = ld8(wp[i] + (size_t)ks * 512);
#pragma unroll
    for (int j = 0; j < TJ; ++j) b[j] = ld8(xp[j] + ks * 32);
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
      for (int j = 0; j < TJ; ++j) acc[i][j] = mfma_16x16x32(w[i], b[j], acc[i][j]);
  }
#pragma unroll
  for (int j = 0; j < TJ; ++j) {
    const int t = t0 + j * 16 + r16;
    if (t >= T) continue;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int n = (nt0 + i) * 16 + g * 4;
      if (n >= N) continue;
      const f32x4 s = acc[i][j] * alpha;
      elt* p = frag_tt ? y + frag_offset(t, (int)(h * hy) + n, frag_tt) : y + t * ldy + h * hy + n;
      *reinterpret_cast<eltx4*>(p) = eltx4{(elt)s[0], (elt)s[1], (elt)s[2], (elt)s[3]};
    }
  }
}

#else   // fp32

constexpr int LA_KEYS = 256;
constexpr int LA_DPT = 4;      // output dims per thread
// One workgroup per (token, head, 1024 output dims): scores of 256 keys at a time, one key per thread, online softmax.
__global__ __launch_bounds__(256) void latent_attn_f32_kernel(LatentAttn a) {
  extern __shared__ __align__(16) float fsm[];    // query row
  __shared__ float ps[LA_KEYS], red[4];
  __shared__ int pgs[LA_KEYS / PAGE];
  const int t = blockIdx.x, h = blockIdx.y, d0 = blockIdx.z * 256 * LA_DPT;
  int seq;
  const int ctx = latent_ctx(a, t, seq), qd = a.NB * 32, rd = a.RB * 32;
  const int32_t* bt = a.block_table + (size_t)seq * a.max_blocks;
  for (int d = threadIdx.x; d < qd; d += 256) fsm[d] = a.q[((size_t)t * a.H + h) * qd + d];
  float m = a.sink ? a.sink[h] : -INFINITY, l = a.sink ? 1.f : 0.f, o[LA_DPT] = {};
  for (int j0 = 0; j0 < ctx; j0 += LA_KEYS) {
    __syncthreads();
    if (threadIdx.x < LA_KEYS / PAGE) {
      const int pg = j0 / PAGE + threadIdx.x;
      const int page = pg * PAGE < ctx ? bt[pg] : -1;
      pgs[threadIdx.x] = page < a.n_pages ? page : -1;
    }
    __syncthreads();
    const int j = j0 + threadIdx.x, page = pgs[threadIdx.x / PAGE];
    float s = -INFINITY;
    if (j < ctx && page >= 0) {
      const float* kp = a.cache + (size_t)page * a.NB * 512 + (j % PAGE) * 8;
      float acc = 0.f;
      for (int b = 0; b < a.NB * 4; ++b)
#pragma unroll
        for (int e = 0; e < 8; ++e) acc = fmaf(kp[(size_t)b * 128 + e], fsm[b * 8 + e], acc);
      s = acc * a.scale;
    }
    float mx = wave_max(s);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = mx;
    __syncthreads();
    const float m_new = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float alpha = m == -INFINITY ? 0.f : expf(m - m_new);
    const float p = s == -INFINITY ? 0.f : expf(s - m_new);
    ps[threadIdx.x] = p;
    const float sum = wave_sum(p);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = sum;
    __syncthreads();
    l = l * alpha + ((red[0] + red[1]) + (red[2] + red[3]));
    m = m_new;
#pragma unroll
    for (int u = 0; u < LA_DPT; ++u) {
      const int d = d0 + u * 256 + threadIdx.x;
      o[u] *= alpha;
      if (d >= rd) continue;
      for (int k = 0; k < LA_KEYS && j0 + k < ctx; ++k) {
        const int pg = pgs[k / PAGE];
        if (pg >= 0) o[u] = fmaf(ps[k], a.cache[latent_offset(pg, a.NB, k % PAGE, d)], o[u]);
      }
    }
  }
#pragma unroll
  for (int u = 0; u < LA_DPT; ++u) {
    const int d = d0 + u * 256 + threadIdx.x;
    if (d < rd) a.out[((size_t)t * a.H + h) * rd + d] = l > 0.f ? o[u] / l : 0.f;
  }
}
#endif

#ifndef MLORA_ELT_F32
template <int NRB, int NW>
int launch_latent_attn(const LatentAttn& a, hipStream_t s) {
  const size_t lds = (size_t)a.NB * 1024 + (size_t)NW * 16 * 68 * sizeof(float);
  static const hipError_t configured =               // the attribute is per kernel, set once per process, by one thread
      hipFuncSetAttribute((const void*)latent_attn_kernel<NRB, NW>, hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);
  if (configured != hipSuccess || lds > 96 * 1024)
    return mlora_set_error(MLORA_ERR_UNSUPPORTED, "latent_attn: cannot reserve %zu bytes of LDS", lds);
  const long outer = ((long)a.T * a.splits + 7) / 8 * 8;
  if (outer * a.n_inner > 0x7fffffffL) return mlora_set_error(MLORA_ERR_UNSUPPORTED, "latent_attn: T=%d is too many tokens", a.T);
  hipLaunchKernelGGL((latent_attn_kernel<NRB, NW>), dim3((unsigned)(outer * a.n_inner)), dim3(NW * WAVE), lds, s, a);
  return MLORA_OK;
}
#endif

}  // namespace

extern "C" int mlora_latent_prep(void* q, void* cache, const void* qkv, int ld, int off_rot, int off_c, int off_kr, float gain, const void* c_norm,
                                 float eps, const int32_t* block_table, int max_blocks, const int32_t* tok_seq, const int32_t* tok_pos,
                                 const float* rope_cos, const float* rope_sin, int max_pos, int T, int H, int R, int rot, int n_pages, int n_seq,
                                 void* stream) {
  MLORA_CHECK(q && cache && qkv && block_table && tok_seq && tok_pos && rope_cos && rope_sin, MLORA_ERR_INVALID, "latent_prep: null pointer");
  MLORA_CHECK(T >= 0 && H > 0 && R > 0 && rot > 0 && rot % 2 == 0 && off_rot >= 0 && off_rot + H * rot <= ld && max_blocks > 0 && n_pages > 0 &&
                  n_seq > 0 && max_pos > 0 && (!c_norm || (off_c >= 0 && off_kr >= 0 && off_c + R <= ld && off_kr + rot <= ld)),
              MLORA_ERR_INVALID, "latent_prep: bad shape T=%d H=%d R=%d rot=%d ld=%d", T, H, R, rot, ld);
  if (T == 0) return MLORA_OK;
  LatentPrep a;
  a.qkv = (const elt*)qkv; a.ld = ld; a.off_rot = off_rot; a.off_c = off_c; a.off_kr = off_kr; a.gain = gain; a.eps = eps;
  a.c_norm = (const elt*)c_norm; a.cache = (elt*)cache; a.block_table = block_table; a.max_blocks = max_blocks; a.n_pages = n_pages;
  a.n_seq = n_seq; a.tok_seq = tok_seq; a.tok_pos = tok_pos; a.cos = rope_cos; a.sin = rope_sin; a.max_pos = max_pos;
  a.H = H; a.R = R; a.rot = rot; a.RB = ceil_div(R, 32); a.NB = a.RB + ceil_div(rot, 32); a.q = (elt*)q;
  hipLaunchKernelGGL(latent_prep_kernel, dim3(T), dim3(256), 0, (hipStream_t)stream, a);
  return mlora_launch_status("latent_prep");
}

// shares of the context a launch is cut into for T tokens that see up to `max_ctx` positions each
extern "C" int mlora_latent_attn_splits(int T, int H, int max_ctx) {
#ifdef MLORA_ELT_F32
  return 1;
#else
  if (T <= 0 || H <= 0 || max_ctx <= 0) return 1;
  const long wgs = (long)T * ceil_div(H, 16);
  int s = (int)(512 / wgs);                                       // two workgroups per compute unit ...
  const int by_ctx = max_ctx / (8 * PAGE);                        // ... of at least two pages per wave
  if (s > by_ctx) s = by_ctx;
  if (s > 32) s = 32;
  return s < 1 ? 1 : s;
#endif
}

extern "C" size_t mlora_latent_attn_workspace_bytes(int T, int H, int R, int splits) {
  if (T <= 0 || H <= 0 || R <= 0 || splits <= 1) return 0;
  return (size_t)splits * T * H * ((size_t)ceil_div(R, 32) * 32 + 2) * sizeof(float);
}

extern "C" int mlora_latent_attn(void* out, const void* q, const void* cache, const int32_t* block_table, int max_blocks, const int32_t* tok_seq,
                                 const int32_t* tok_pos, const float* sink, float scale, int T, int H, int R, int rot, int n_pages, int n_seq,
                                 int splits, void* workspace, size_t workspace_bytes, void* stream) {
  MLORA_CHECK(out && q && cache && block_table && tok_seq && tok_pos, MLORA_ERR_INVALID, "latent_attn: null pointer");
  MLORA_CHECK(T >= 0 && H > 0 && H <= 65535 && R > 0 && rot > 0 && max_blocks > 0 && n_pages > 0 && n_seq > 0 && splits >= 1, MLORA_ERR_INVALID,
              "latent_attn: bad shape T=%d H=%d R=%d rot=%d", T, H, R, rot);
  if (T == 0) return MLORA_OK;
  LatentAttn a;
  a.out = (elt*)out; a.q = (const elt*)q; a.cache = (const elt*)cache; a.block_table = block_table; a.max_blocks = max_blocks;
  a.n_pages = n_pages; a.n_seq = n_seq; a.tok_seq = tok_seq; a.tok_pos = tok_pos; a.sink = sink; a.scale = scale;
  a.T = T; a.H = H; a.RB = ceil_div(R, 32); a.NB = a.RB + ceil_div(rot, 32); a.splits = splits;
  a.part_o = a.part_ml = nullptr; a.n_inner = a.chunks = 1;
  hipStream_t s = (hipStream_t)stream;
#ifdef MLORA_ELT_F32
  MLORA_CHECK(splits == 1 && a.NB * 128 <= 48 * 1024, MLORA_ERR_UNSUPPORTED, "latent_attn: splits=%d R=%d not served in fp32", splits, R);
  hipLaunchKernelGGL(latent_attn_f32_kernel, dim3(T, H, ceil_div(a.RB * 32, 256 * LA_DPT)), dim3(256), a.NB * 128, s, a);
#else
  if (splits > 1) {
    MLORA_CHECK(workspace && workspace_bytes >= mlora_latent_attn_workspace_bytes(T, H, R, splits), MLORA_ERR_WORKSPACE,
                "latent_attn: workspace of %zu bytes needed", mlora_latent_attn_workspace_bytes(T, H, R, splits));
    a.part_o = (float*)workspace;
    a.part_ml = a.part_o + (size_t)splits * T * H * a.RB * 32;
  }
  const int nrb = a.RB <= 2 ? 2 : a.RB <= 4 ? 4 : a.RB <= 8 ? 8 : 16;
  a.chunks = ceil_div(a.RB, nrb);
  a.n_inner = ceil_div(H, 16) * a.chunks;
  int e;
  if (nrb == 2) e = launch_latent_attn<2, 4>(a, s);
  else if (nrb == 4) e = launch_latent_attn<4, 4>(a, s);
  else if (nrb == 8) e = launch_latent_attn<8, 4>(a, s);
  else e = launch_latent_attn<16, 4>(a, s);
  if (e) return e;
  if (splits > 1) {
    MLORA_CHECK((long)T * H <= 0x7fffffffL, MLORA_ERR_UNSUPPORTED, "latent_attn: T=%d is too many tokens", T);
    hipLaunchKernelGGL(latent_merge_kernel, dim3(T * H), dim3(128), 0, s, a);
  }
#endif
  return mlora_launch_status("latent_attn");
}

#ifndef MLORA_ELT_F32
extern "C" int mlora_head_linear(void* y, int y_layout, long ldy, long head_y, const void* x, long ldx, long head_x, const void* W, int heads, int T,
                                 int K, int N, float alpha, void* stream) {
  MLORA_CHECK(y && x && W, MLORA_ERR_INVALID, "head_linear: null pointer");
  MLORA_CHECK(T >= 0 && heads > 0 && heads <= 65535 && K > 0 && K % 32 == 0 && N > 0 && N % 16 == 0 && ldx % 8 == 0 && head_x % 8 == 0 &&
                  head_y % 4 == 0 && (y_layout == MLORA_FRAG ? (heads * head_y) % 32 == 0 : ldy % 4 == 0) && ceil_div(T, 16) <= 65535,
              MLORA_ERR_UNSUPPORTED, "head_linear: need K %% 32 == 0, N %% 16 == 0 and aligned rows (T=%d K=%d N=%d)", T, K, N);
  if (T == 0) return MLORA_OK;
  const int tt = y_layout == MLORA_FRAG ? mlora_frag_tiles(T) : 0;
  hipStream_t s = (hipStream_t)stream;
#define MLORA_HL(NI, TJ)                                                                                                              \
  hipLaunchKernelGGL((head_linear_kernel<NI, TJ>), dim3(ceil_div(N, 64 * NI), ceil_div(T, 16 * TJ), heads), dim3(256), 0, s, (elt*)y, \
                     ldy, head_y, tt, (const elt*)x, ldx, head_x, (const elt*)W, T, K, N, alpha)
  if (T <= 16) MLORA_HL(1, 1);
  else if (T <= 32) MLORA_HL(1, 2);
  else if (T <= 256) MLORA_HL(1, 4);
  else MLORA_HL(4, 4);
#undef MLORA_HL
  return mlora_launch_status("head_linear");
}
#endif
