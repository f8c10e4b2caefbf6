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
//
// Tied attention (TIED): the heads of a group share a key/value head whose values are its keys before their norm.  A page
// holds the values v of each of the G key/value heads, [n_pages, G, RB, 4, 16, 8], and one number per token and head,
// 1 / rms(v) [n_pages, G, 16] fp32, so that a key is (1 / rms) v w and is never stored: the norm's weight w goes to the queries,
// the number to the scores.  A distance bias slope_h (i - j) is taken off the scores.
// Normed keys have a root mean square of at most one, so a score lies within B = |scale| |q| sqrt(D) of zero, and the query's own key
// (distance 0) scores at least -B: a key whose bias exceeds 2 B by 126 bits has a weight that fp32 holds as zero.  Pages behind that
// reach are not read.
#include <type_traits>

#include "common.h"

// Every kernel with matrix-core products here names its waves per SIMD (two) in its launch bounds: without, the compiler
// keeps the accumulators in the accumulation registers and has been seen to read them back before a loop's last product
// had written them.
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
  elt* q;                   // the rotated query parts: row (t, h) at (t H + h) q_ld + q_off, padded to whole blocks
  int q_ld, q_off;
};

// One workgroup per token: rotates the heads' query parts into the query rows (their `gain` is left to the scores' scale),
// norms the latent, rotates the shared key part and stores both in the token's page slot.  Neighbouring elements (2 i, 2 i + 1) turn by the table's angle i.
__device__ __forceinline__ void latent_prep(const LatentPrep& a, int t, float* __restrict__ red) {
  const int seq = a.tok_seq[t], pos = a.tok_pos[t];
  if (seq < 0 || seq >= a.n_seq || pos < 0 || pos >= a.max_pos || pos / PAGE >= a.max_blocks) return;   // uniform
  const elt* row = a.qkv + (size_t)t * a.ld;
  const int half = a.rot / 2, rp = (a.NB - a.RB) * 32;
  const float* cp = a.cos + (size_t)pos * half;
  const float* sp = a.sin + (size_t)pos * half;
  elt* q = a.q + (size_t)t * a.H * a.q_ld + a.q_off;
  for (int i = threadIdx.x; i < a.H * (rp / 2); i += 256) {
    const int h = i / (rp / 2), k = i - h * (rp / 2);
    float u = 0.f, v = 0.f;
    if (k < half) {
      const float x1 = (float)row[a.off_rot + h * a.rot + 2 * k], x2 = (float)row[a.off_rot + h * a.rot + 2 * k + 1];
      u = x1 * cp[k] - x2 * sp[k];
      v = x2 * cp[k] + x1 * sp[k];
    }
    *reinterpret_cast<eltx2*>(q + (size_t)h * a.q_ld + 2 * k) = eltx2{(elt)u, (elt)v};
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

__global__ __launch_bounds__(256) void latent_prep_kernel(LatentPrep a) {
  __shared__ float red[4];
  latent_prep(a, blockIdx.x, red);
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
  const float* key_scale;   // tied: [n_pages, G, 16]
  const float* slopes;      // tied: [H]
  int G, gs, gt, D;         // tied: key/value heads, heads per group, 16-head tiles per group, columns of a head
  int frag_tt;              // `out` in fragment order (tied) if > 0
};

__device__ __forceinline__ size_t latent_out_offset(const LatentAttn& a, int t, int h, int d) {
  return a.frag_tt ? frag_offset(t, h * a.RB * 32 + d, a.frag_tt) : ((size_t)t * a.H + h) * (a.RB * 32) + d;
}

// the context a token sees: every position up to its own
__device__ __forceinline__ int latent_ctx(const LatentAttn& a, int t, int& seq) {
  seq = a.tok_seq[t];
  int ctx = a.tok_pos[t] + 1;
  if (seq < 0 || seq >= a.n_seq || ctx < 0) ctx = 0;
  if (seq < 0 || seq >= a.n_seq) seq = 0;
  return ctx < a.max_blocks * PAGE ? ctx : a.max_blocks * PAGE;
}

// tied: positions behind a query that can have a weight, given the square of its length (see above)
__device__ __forceinline__ float tied_reach(float qq, int D, float scale, float slope) {
  const float B = fabsf(scale) * sqrtf(qq * (float)D) * 1.02f;      // a margin for the rounding of queries and keys
  return fminf((2.f * B + 90.f) / fmaxf(slope, 1e-30f), 1e9f) + 2.f;
}

#ifndef MLORA_ELT_F32
// A workgroup takes one token, 16 heads (the columns of the matrix-core tiles), a share of the context (split) and up to
// NRB blocks of the latent as output (chunk; all of it up to NRB blocks).  A wave takes every NW-th page:
//   S^T = K . Q^T        the page's fragments as they lie in the cache, queries from LDS
//   page^T               two products with halves of the identity per 32 dims: exact
//   O^T += page^T . P^T  P as hi + lo halves in the two halves of the k-slots, the page's values repeated in both
// The waves' states (m, l, O) meet in LDS, 64 dims at a time.
template <int NRB, int NW, bool TIED = false>
__global__ __launch_bounds__(NW * WAVE, 2) void latent_attn_kernel(LatentAttn a) {
  extern __shared__ __align__(16) char smem_raw[];
  const int RBp = a.chunks * NRB, KR = TIED ? 0 : a.NB - a.RB, KRp = TIED ? 0 : KR > 2 ? KR : 2;   // blocks in LDS: the latent's, the rotated part's
  elt* qs = reinterpret_cast<elt*>(smem_raw);                        // [RBp + KRp][64][8] query fragments, zero where there is no block
  float* sacc = reinterpret_cast<float*>(qs + (RBp + KRp) * 512);    // [NW][16][68]
  __shared__ float sm[NW][16], sl[NW][16];
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int col = lane & 15, g = lane >> 4;
  // the workgroups that walk the same pages (inner index: head groups and chunks) run on one XCD
  const int x8 = blockIdx.x & 7, rest = blockIdx.x >> 3;
  const int inner = rest % a.n_inner, outer = (rest / a.n_inner) * 8 + x8;
  if (outer >= a.T * a.splits) return;                               // uniform
  const int t = outer / a.splits, split = outer - t * a.splits;
  const int hg = inner / a.chunks, b0 = (inner - hg * a.chunks) * NRB;
  // the heads of the tile's columns: h0 .. h0 + hn - 1
  const int kvh = TIED ? hg / a.gt : 0, hw = TIED ? (hg - kvh * a.gt) * 16 : hg * 16;
  const int h0 = TIED ? kvh * a.gs + hw : hw, hn = (TIED ? a.gs : a.H) - hw;
  int seq;
  const int ctx = latent_ctx(a, t, seq);
  const int npages = (ctx + PAGE - 1) / PAGE;
  int per = (npages + a.splits - 1) / a.splits;
  int p0 = split * per, p1 = p0 + per < npages ? p0 + per : npages;
  const int32_t* __restrict__ bt = a.block_table + (size_t)seq * a.max_blocks;
  const int qd = a.NB * 32;

  for (int i = threadIdx.x; i < (RBp + KRp) * 64; i += NW * WAVE) {
    const int slot = i >> 6, l = i & 63, h = h0 + (l & 15);
    const int kb = slot < RBp ? slot : slot - RBp + a.RB;
    eltx8 v = eltx8{0, 0, 0, 0, 0, 0, 0, 0};
    if ((l & 15) < hn && (slot < RBp ? kb < a.RB : kb < a.NB)) v = ld8(a.q + ((size_t)t * a.H + h) * qd + kb * 32 + (l >> 4) * 8);
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
  const float slope = TIED ? a.slopes[h0 + (col < hn ? col : 0)] : 0.f;
  if constexpr (TIED) {                                              // the pages within reach of any of the heads
    float qq = 0.f;
    for (int s = 0; s < RBp; ++s) {
      const eltx8 v = ld8(qs + (s * 64 + lane) * 8);
#pragma unroll
      for (int e = 0; e < 8; ++e) qq = fmaf((float)v[e], (float)v[e], qq);
    }
    qq += __shfl_xor(qq, 16, WAVE);
    qq += __shfl_xor(qq, 32, WAVE);
    const float reach = wave_max(col < hn ? tied_reach(qq, a.D, a.scale, slope) : 0.f);
    const int back = (int)fminf(reach, (float)ctx);
    const int pb = __builtin_amdgcn_readfirstlane((ctx - back > 0 ? ctx - back : 0) / PAGE);
    per = (npages - pb + a.splits - 1) / a.splits;
    p0 = pb + split * per;
    p1 = p0 + per < npages ? p0 + per : npages;
  }

  float m = -INFINITY, l = 0.f;
  f32x4 O[2 * NRB];
#pragma unroll
  for (int db = 0; db < 2 * NRB; ++db) O[db] = f32x4{0.f, 0.f, 0.f, 0.f};

  // the cache page of the context's page pg (page 0 for one outside the cache: every key of it is masked)
  auto page_of = [&](int pg, bool& ok) {
    const int page = bt[pg];
    ok = page >= 0 && page < a.n_pages;
    return a.cache + ((size_t)(ok ? page : 0) * (TIED ? a.G : 1) + kvh) * a.NB * 512 + lane * 8;
  };
  // tied: the scale of this lane's four keys of a page, and its head's slope
  auto scale_of = [&](int pg) {
    const int page = bt[pg];
    return *reinterpret_cast<const f32x4*>(a.key_scale + ((size_t)(page >= 0 && page < a.n_pages ? page : 0) * a.G + kvh) * PAGE + 4 * g);
  };
  f32x4 ksc = f32x4{0.f, 0.f, 0.f, 0.f};
  eltx8 kf[NRB], rf[2];
  bool ok = false, ok_next = false;
  const elt* kp = a.cache;
  if (p0 + wave < p1) {
    kp = page_of(p0 + wave, ok);
#pragma unroll
    for (int b = 0; b < NRB; ++b) kf[b] = ld8(kp + (b0 + b < a.RB ? b0 + b : a.RB - 1) * 512);
    if constexpr (TIED) {
      ksc = scale_of(p0 + wave);
    } else {
#pragma unroll
      for (int r = 0; r < 2; ++r) rf[r] = ld8(kp + (r < KR ? a.RB + r : a.RB) * 512);
    }
  }
  for (int pg = p0 + wave; pg < p1; pg += NW) {
    // the next page's fragments are requested one by one as this page's are done with
    const elt* kn = page_of(pg + NW < p1 ? pg + NW : pg, ok_next);
    // two chains of products: st[r] = S[token 4 g + r][head col].  A block that does not exist meets zero queries.
    f32x4 st = f32x4{0.f, 0.f, 0.f, 0.f}, st1 = st, ksn = st;
    if constexpr (TIED) {
      ksn = scale_of(pg + NW < p1 ? pg + NW : pg);
    } else {
      st = mfma_16x16x32(rf[0], ld8(qs + (RBp * 64 + lane) * 8), f32x4{0.f, 0.f, 0.f, 0.f});
      st1 = mfma_16x16x32(rf[1], ld8(qs + ((RBp + 1) * 64 + lane) * 8), f32x4{0.f, 0.f, 0.f, 0.f});
      rf[0] = ld8(kn + a.RB * 512);
      rf[1] = ld8(kn + (KR > 1 ? a.RB + 1 : a.RB) * 512);
    }
#pragma unroll
    for (int b = 0; b < NRB; b += 2) {
      st = mfma_16x16x32(kf[b], ld8(qs + ((b0 + b) * 64 + lane) * 8), st);
      st1 = mfma_16x16x32(kf[b + 1], ld8(qs + ((b0 + b + 1) * 64 + lane) * 8), st1);
    }
    for (int r = 2; r < KR; ++r) st = mfma_16x16x32(ld8(kp + (a.RB + r) * 512), ld8(qs + ((RBp + r) * 64 + lane) * 8), st);
    if (a.chunks > 1)                                                // the latent's blocks outside this chunk
      for (int kb = 0; kb < a.RB; ++kb)
        if (kb < b0 || kb >= b0 + NRB) st = mfma_16x16x32(ld8(kp + kb * 512), ld8(qs + (kb * 64 + lane) * 8), st);
    st += st1;

    float pm = -INFINITY;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int j = pg * PAGE + 4 * g + r;
      const float sc = TIED ? fmaf(-slope, (float)(ctx - 1 - j), st[r] * a.scale * ksc[r]) : st[r] * a.scale;
      st[r] = !ok || j >= ctx ? -INFINITY : sc;
      pm = fmaxf(pm, st[r]);
    }
    pm = fmaxf(pm, __shfl_xor(pm, 16, WAVE));
    pm = fmaxf(pm, __shfl_xor(pm, 32, WAVE));
    const float m_new = fmaxf(m, pm);
    if (__any(m_new > m)) {                                          // uniform: the maximum rarely moves after the first pages
      const float alpha = m == -INFINITY ? 0.f : __expf(m - m_new);
      l *= alpha;
#pragma unroll
      for (int db = 0; db < 2 * NRB; ++db) O[db] *= alpha;
      m = m_new;
    }
    const float mm = m == -INFINITY ? 0.f : m;
    eltx8 pa;
    float ps = 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float p = __expf(st[r] - mm);
      ps += p;
      const elt hi = (elt)p;
      pa[r] = hi;
      pa[4 + r] = (elt)(p - (float)hi);
    }
    l += ps;                                                         // the lane's share of its column's sum
#pragma unroll
    for (int b = 0; b < NRB; ++b) {
      const f32x4 t0 = mfma_16x16x32(kf[b], id0, f32x4{0.f, 0.f, 0.f, 0.f}), t1 = mfma_16x16x32(kf[b], id1, f32x4{0.f, 0.f, 0.f, 0.f});
      asm volatile("" ::: "memory");                                 // not earlier: the request goes into the registers just read
      kf[b] = ld8(kn + (b0 + b < a.RB ? b0 + b : a.RB - 1) * 512);
      const eltx4 h0 = eltx4{(elt)t0[0], (elt)t0[1], (elt)t0[2], (elt)t0[3]}, h1 = eltx4{(elt)t1[0], (elt)t1[1], (elt)t1[2], (elt)t1[3]};
      O[2 * b] = mfma_16x16x32(eltx8{h0[0], h0[1], h0[2], h0[3], h0[0], h0[1], h0[2], h0[3]}, pa, O[2 * b]);   // O^T[dim 32 b + 4 g + r][head col]
      O[2 * b + 1] = mfma_16x16x32(eltx8{h1[0], h1[1], h1[2], h1[3], h1[0], h1[1], h1[2], h1[3]}, pa, O[2 * b + 1]);
    }
    kp = kn;
    ok = ok_next;
    ksc = ksn;
  }
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  if (g == 0) {
    sm[wave][col] = m;
    sl[wave][col] = l;
  }
  __syncthreads();
  // per head, once: what every wave's sums are multiplied with, and (M, L)
  if (threadIdx.x < 16) {
    const int hc = threadIdx.x, h = h0 + hc;
    const float sk = !TIED && a.splits == 1 && a.sink && hc < hn ? a.sink[h] : -INFINITY;
    float M = sk, L = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) M = fmaxf(M, sm[w][hc]);
    if (sk != -INFINITY) L = __expf(sk - M);
    float f[NW];
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      f[w] = sm[w][hc] == -INFINITY ? 0.f : __expf(sm[w][hc] - M);
      L += sl[w][hc] * f[w];
    }
    const float inv = a.splits > 1 ? 1.f : L > 0.f ? 1.f / L : 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) sm[w][hc] = f[w] * inv;
    if (a.splits > 1 && hc < hn && b0 == 0) {
      const size_t r = ((size_t)split * a.T + t) * a.H + h;
      a.part_ml[2 * r] = M;
      a.part_ml[2 * r + 1] = L;
    }
  }
#pragma unroll
  for (int c = 0; c < NRB; c += 2) {                                 // 64 dims
    if (b0 + c < a.RB) {                                             // uniform
      __syncthreads();
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (2 * c + u < 2 * NRB) *reinterpret_cast<f32x4*>(sacc + (wave * 16 + col) * 68 + u * 16 + 4 * g) = O[(2 * c + u) % (2 * NRB)];
      __syncthreads();
      for (int e = threadIdx.x; e < 16 * 16; e += NW * WAVE) {
        const int hc = e >> 4, dd = (e & 15) * 4, h = h0 + hc, d = (b0 + c) * 32 + dd;
        if (hc >= hn || d >= a.RB * 32 || d >= (b0 + NRB) * 32) continue;
        f32x4 o = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < NW; ++w) o += *reinterpret_cast<const f32x4*>(sacc + (w * 16 + hc) * 68 + dd) * sm[w][hc];
        if (a.splits == 1)
          *reinterpret_cast<eltx4*>(a.out + (TIED ? latent_out_offset(a, t, h, d) : ((size_t)t * a.H + h) * (a.RB * 32) + d)) =
              eltx4{(elt)o[0], (elt)o[1], (elt)o[2], (elt)o[3]};
        else
          *reinterpret_cast<f32x4*>(a.part_o + (((size_t)split * a.T + t) * a.H + h) * (a.RB * 32) + d) = o;
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
    *reinterpret_cast<eltx4*>(a.out + latent_out_offset(a, th / a.H, h, d)) = eltx4{(elt)(o[0] * inv), (elt)(o[1] * inv), (elt)(o[2] * inv), (elt)(o[3] * inv)};
  }
}

// ---------------------------------------------------------------------------------------------
// Prompts: with many queries per key it is cheaper to make the heads' keys and values once than to work on the latents
// (dim + rot_dim + vdim products per score instead of 2 kv_rank + rot_dim).  The keys and values of the contexts of a pass are
// written to scratch memory in the order the matrix cores read them, one context after the other, each padded to whole
// blocks of 64 keys with zeros:
//   K [H, pages, KN, 512]      a page's fragments (16 tokens x 32 dims), as in a cache page
//   V [H, pages / 2, VB, 512]  16 dims x 32 tokens: lane (dim % 16, g) holds tokens 4 g .. + 3 of the even, then of the odd page
//   R [pages, KR, 512]         the rotated key part, shared by the heads
// ---------------------------------------------------------------------------------------------
struct LatentExpand {
  elt* k;
  elt* v;
  elt* r;
  const elt* cache;
  const int32_t* phys;      // [pages] cache page of a scratch page, -1: padding
  const elt* uk;            // packed [H * KN * 32, RB * 32]
  const elt* uv;            // packed [H * VB * 16, RB * 32]
  int pages, n_pages, H, RB, KR, KN, VB;
  int kb_blocks, vb_blocks; // workgroups along x that make keys, then values; one more copies R
};

// A wave makes 16 LE_ROWS rows (of W_uk or W_uv) x 4 pages; the two halves of a workgroup take the same rows for neighbouring
// pages, so that a weight fragment crosses from the second-level cache once for both.
constexpr int LE_ROWS = 4;
__global__ __launch_bounds__(512, 3) void latent_expand_kernel(LatentExpand a) {
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int pg0 = blockIdx.y * 8 + (wave >> 2) * 4, NB = a.RB + a.KR;
  if (pg0 >= a.pages) return;                                        // no barrier below
  int page[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    page[j] = a.phys[pg0 + j];
    if (page[j] >= a.n_pages) page[j] = -1;
  }
  const eltx8 zero = eltx8{0, 0, 0, 0, 0, 0, 0, 0};
  int bx = blockIdx.x;
  if (bx > a.kb_blocks + a.vb_blocks) return;
  if (bx == a.kb_blocks + a.vb_blocks) {
    for (int i = threadIdx.x & 255; i < 4 * a.KR * 64; i += 256) {
      const int j = i / (a.KR * 64), o = i - j * (a.KR * 64);
      const int pj = a.phys[pg0 + j];
      st8(a.r + ((size_t)(pg0 + j) * a.KR * 64 + o) * 8,
          pj >= 0 && pj < a.n_pages ? ld8(a.cache + (size_t)pj * NB * 512 + a.RB * 512 + o * 8) : zero);
    }
    return;
  }
  const bool val = bx >= a.kb_blocks;                                // uniform
  if (val) bx -= a.kb_blocks;
  const int tiles = val ? a.H * a.VB : a.H * a.KN * 2;
  const int nt0 = (bx * 4 + (wave & 3)) * LE_ROWS;
  if (nt0 >= tiles) return;
  const elt* wp = (val ? a.uv : a.uk) + lane * 8;
  int wo[LE_ROWS];                                                   // uniform
  const elt* cp[4];
#pragma unroll
  for (int i = 0; i < LE_ROWS; ++i) wo[i] = (nt0 + i < tiles ? nt0 + i : tiles - 1) * a.RB * 512;
#pragma unroll
  for (int i = 0; i < 4; ++i) cp[i] = a.cache + (size_t)(page[i] >= 0 ? page[i] : 0) * NB * 512 + lane * 8;
  f32x4 acc[LE_ROWS][4];
#pragma unroll
  for (int i = 0; i < LE_ROWS; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  auto products = [&](auto V) {
    eltx8 w[LE_ROWS], c[4];
#pragma unroll
    for (int i = 0; i < LE_ROWS; ++i) w[i] = ld8(wp + wo[i]);
#pragma unroll
    for (int i = 0; i < 4; ++i) c[i] = ld8(cp[i]);
    for (int kb = 1; kb <= a.RB; ++kb) {
      const int kc = kb < a.RB ? kb : 0;                             // the last prefetch wraps to a valid address and is discarded
      eltx8 wn[LE_ROWS], cn[4];
#pragma unroll
      for (int i = 0; i < LE_ROWS; ++i) wn[i] = ld8(wp + (wo[i] + kc * 512));
#pragma unroll
      for (int i = 0; i < 4; ++i) cn[i] = ld8(cp[i] + kc * 512);
      __builtin_amdgcn_sched_barrier(0);                             // the requests go out ahead of the products
#pragma unroll
      for (int i = 0; i < LE_ROWS; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = decltype(V)::value ? mfma_16x16x32(c[j], w[i], acc[i][j]) : mfma_16x16x32(w[i], c[j], acc[i][j]);
#pragma unroll
      for (int i = 0; i < LE_ROWS; ++i) w[i] = wn[i];
#pragma unroll
      for (int i = 0; i < 4; ++i) c[i] = cn[i];
    }
  };
  if (val) products(std::true_type());
  else products(std::false_type());
  const int r16 = lane & 15, g = lane >> 4;
#pragma unroll
  for (int i = 0; i < LE_ROWS; ++i) {
    const int nt = nt0 + i;
    if (nt >= tiles) continue;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const f32x4 s = page[j] >= 0 ? acc[i][j] : f32x4{0.f, 0.f, 0.f, 0.f};
      const eltx4 o = eltx4{(elt)s[0], (elt)s[1], (elt)s[2], (elt)s[3]};
      if (val) {                                                     // s[r] = token 4 g + r, dim r16 of the tile
        const int h = nt / a.VB, db = nt - h * a.VB, p = pg0 + j;
        *reinterpret_cast<eltx4*>(a.v + (((size_t)h * (a.pages / 2) + p / 2) * a.VB + db) * 512 + lane * 8 + (p & 1) * 4) = o;
      } else {                                                       // s[r] = dim 4 g + r of the tile, token r16
        const int h = nt / (2 * a.KN), d = (nt - h * 2 * a.KN) * 16 + g * 4;
        *reinterpret_cast<eltx4*>(a.k + (((size_t)h * a.pages + pg0 + j) * a.KN + (d >> 5)) * 512 + ((d >> 3) & 3) * 128 + r16 * 8 + (d & 7)) = o;
      }
    }
  }
}

struct LatentPrefill {
  elt* out;                 // [T, H * VB * 16], row-major (frag_tt == 0: row stride ld_out) or in fragment order
  int frag_tt, ld_out;
  const elt* q;             // [T, ld_q]: the heads' unrotated query parts at h * KN * 32
  int ld_q;
  const elt* qr;            // [T, H, KR * 32]: their rotated parts
  const elt* k;
  const elt* v;
  const elt* r;
  const int4* tiles;        // {first token, tokens, first scratch page, position of the first token}, long key ranges first
  const float* sink;
  float scale;
  int H, pages, KN, KR, VB;
  const float* slopes;      // tied: [H]
  int gs, D;                // tied: heads per key/value head, columns of a head
};

// Four waves own up to 128 consecutive queries of one head of one sequence, a wave 32 of them as two 16-query tiles.  Keys are
// walked in blocks of 64: K and V go from scratch memory straight into LDS, double buffered, one bare barrier per block.
// S^T = K . Q^T, softmax state per lane (its own query column), O^T += V^T . P^T with P as hi + lo halves.
// KB = KN + KR and VB bound the register arrays; EXACT: they are the sizes themselves.
constexpr int LP_WAVES = 4;
constexpr int LP_QT = 2;
constexpr int LP_TOK = LP_WAVES * LP_QT * 16;
// TIED: the heads of a group read one K and V (no rotated part), and a distance bias is taken off the scores.
template <int KB_, int VB_, bool EXACT, bool TIED = false>
__global__ __launch_bounds__(LP_WAVES* WAVE, 2) void latent_prefill_kernel(LatentPrefill a) {
  extern __shared__ __align__(16) elt lsm[];                         // [2][4 KB + 2 VB][512]
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int qi = lane & 15, g = lane >> 4;
  const int KN = TIED && EXACT ? KB_ : a.KN, KR = TIED ? 0 : a.KR, KB = EXACT ? KB_ : KN + KR, VB = EXACT ? VB_ : a.VB;
  const int PIECES = 4 * KB + 2 * VB;                                // 1 KiB pieces of a key block
  // tied: the long ranges are those of the heads with small slopes, which the tiles take to another XCD each time
  const int h = TIED ? (blockIdx.x + blockIdx.y) % gridDim.x : blockIdx.x;
  const int4 tile = a.tiles[blockIdx.y];
  const int wq = wave * LP_QT * 16;                                  // this wave's first query of the tile
  eltx8 qf[LP_QT][KB_];
#pragma unroll
  for (int u = 0; u < LP_QT; ++u) {
    const int i = wq + u * 16 + qi;
    const size_t t = tile.x + (i < tile.y ? i : tile.y - 1);
#pragma unroll
    for (int kb = 0; kb < KB_; ++kb) {
      qf[u][kb] = eltx8{0, 0, 0, 0, 0, 0, 0, 0};
      if (kb < KB) qf[u][kb] = kb < KN ? ld8(a.q + t * a.ld_q + (h * KN + kb) * 32 + g * 8) : ld8(a.qr + (t * a.H + h) * (KR * 32) + (kb - KN) * 32 + g * 8);
    }
  }
  const float c2 = a.scale * 1.44269504088896340736f;                // softmax in base 2
  float m[LP_QT], l[LP_QT];
  f32x4 O[LP_QT][VB_];
#pragma unroll
  for (int u = 0; u < LP_QT; ++u) {
    m[u] = -INFINITY;
    l[u] = 0.f;
#pragma unroll
    for (int db = 0; db < VB_; ++db) O[u][db] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const int last = tile.w + tile.y - 1;                              // position of the tile's last query
  const int nblk = last / 64 + 1;
  const int kvh = TIED ? h / a.gs : h;
  const float slope = TIED ? a.slopes[h] * 1.44269504088896340736f : 0.f;
  const elt* kh = a.k + ((size_t)kvh * a.pages + tile.z) * KN * 512 + lane * 8;
  const elt* vh = a.v + ((size_t)kvh * (a.pages / 2) + tile.z / 2) * VB * 512 + lane * 8;
  const elt* rh = a.r + (size_t)tile.z * KR * 512 + lane * 8;
  // piece i of a block: page p = i / KB, fragment i % KB of it for i < 4 KB; then the pairs' V pieces
  auto issue = [&](int b) {
    elt* dst = lsm + (b & 1) * PIECES * 512;
    for (int i = wave; i < PIECES; i += LP_WAVES) {                  // uniform
      const elt* src;
      if (i < 4 * KB) {
        const int p = i / KB, f = i - p * KB;
        src = f < KN ? kh + ((size_t)(4 * b + p) * KN + f) * 512 : rh + ((size_t)(4 * b + p) * KR + f - KN) * 512;
      } else {
        src = vh + ((size_t)(2 * b) * VB + i - 4 * KB) * 512;
      }
      __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)src,
                                       (__attribute__((address_space(3))) void*)(dst + i * 512), 16, 0, 0);
    }
  };
  int b0 = 0;
  if constexpr (TIED) {                                              // the first block within reach of any of the queries
    __shared__ float qmax[LP_WAVES];
    float qq = 0.f;
#pragma unroll
    for (int u = 0; u < LP_QT; ++u) {
      float s = 0.f;
#pragma unroll
      for (int kb = 0; kb < KB_; ++kb)
#pragma unroll
        for (int e = 0; e < 8; ++e) s = fmaf((float)qf[u][kb][e], (float)qf[u][kb][e], s);
      s += __shfl_xor(s, 16, WAVE);
      s += __shfl_xor(s, 32, WAVE);
      qq = fmaxf(qq, s);
    }
    qq = wave_max(qq);
    if (lane == 0) qmax[wave] = qq;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < LP_WAVES; ++i) qq = fmaxf(qq, qmax[i]);
    const int back = (int)fminf(tied_reach(qq, a.D, a.scale, a.slopes[h]), (float)(tile.w + 1));
    b0 = __builtin_amdgcn_readfirstlane((tile.w - back > 0 ? tile.w - back : 0) / 64);
  }
  issue(b0);
  for (int b = b0; b < nblk; ++b) {
    asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");      // this wave's pieces of block b have landed, its reads of b - 1 are done
    bare_barrier();
    if (b + 1 < nblk) issue(b + 1);                                  // into the buffer of block b - 1
    const elt* ks = lsm + (b & 1) * PIECES * 512 + lane * 8;
    const elt* vs = ks + 4 * KB * 512;
    bool act[LP_QT];                                                 // uniform: the 16-query tile exists and reaches the block
#pragma unroll
    for (int u = 0; u < LP_QT; ++u) {
      const int i1 = wq + u * 16 + 15 < tile.y - 1 ? wq + u * 16 + 15 : tile.y - 1;
      act[u] = wq + u * 16 < tile.y && tile.w + i1 >= b * 64;
    }
    if (!act[0] && !act[1]) continue;
    f32x4 st[LP_QT][4];                                              // st[u][p][r] = S[key 4 g + r of page p][query qi of tile u]
#pragma unroll
    for (int p = 0; p < 4; ++p) {
#pragma unroll
      for (int u = 0; u < LP_QT; ++u) st[u][p] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kb = 0; kb < KB_; ++kb) {
        if (EXACT || kb < KB) {
          const eltx8 kf = ld8(ks + (p * KB + kb) * 512);
#pragma unroll
          for (int u = 0; u < LP_QT; ++u) st[u][p] = mfma_16x16x32(kf, qf[u][kb], st[u][p]);
        }
      }
    }
    eltx8 ph[LP_QT][2], pl[LP_QT][2];
#pragma unroll
    for (int u = 0; u < LP_QT; ++u) {
      const int lim = tile.w + wq + u * 16 + qi - b * 64 - 4 * g;    // key (p, r) of this lane is visible while 16 p + r <= lim
      float pm = -INFINITY;
#pragma unroll
      for (int p = 0; p < 4; ++p) {
        if constexpr (TIED) {
          const float off = slope * (float)(p * 16 - lim);           // minus the slope times the distance of the lane's first key of the page
#pragma unroll
          for (int r = 0; r < 4; ++r) st[u][p][r] = fmaf(st[u][p][r], c2, off + slope * r);
        } else {
          st[u][p] *= c2;
        }
      }
      if (tile.w + wq + u * 16 < b * 64 + 63) {                      // uniform: the block crosses the tile's diagonal
#pragma unroll
        for (int p = 0; p < 4; ++p)
#pragma unroll
          for (int r = 0; r < 4; ++r) st[u][p][r] = p * 16 + r <= lim ? st[u][p][r] : -INFINITY;
      }
#pragma unroll
      for (int p = 0; p < 4; ++p)
#pragma unroll
        for (int r = 0; r < 4; ++r) pm = fmaxf(pm, st[u][p][r]);
      pm = fmaxf(pm, __shfl_xor(pm, 16, WAVE));
      pm = fmaxf(pm, __shfl_xor(pm, 32, WAVE));
      const float mn = fmaxf(m[u], pm);
      if (__any(mn > m[u])) {                                        // uniform
        const float alpha = m[u] == -INFINITY ? 0.f : exp2f(m[u] - mn);
        l[u] *= alpha;
#pragma unroll
        for (int db = 0; db < VB_; ++db) O[u][db] *= alpha;
        m[u] = mn;
      }
      const float mm = mn == -INFINITY ? 0.f : mn;                   // a query that sees nothing of this block yet (m stays -inf)
      float ps = 0.f;
#pragma unroll
      for (int p = 0; p < 4; ++p)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float e = __builtin_amdgcn_exp2f(st[u][p][r] - mm);
          ps += e;
          const elt hi = (elt)e;
          ph[u][p >> 1][(p & 1) * 4 + r] = hi;
          pl[u][p >> 1][(p & 1) * 4 + r] = (elt)(e - (float)hi);
        }
      l[u] += ps;
    }
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int db = 0; db < VB_; ++db) {
        if (EXACT || db < VB) {
          const eltx8 vf = ld8(vs + (j * VB + db) * 512);
#pragma unroll
          for (int u = 0; u < LP_QT; ++u) {
            O[u][db] = mfma_16x16x32(vf, ph[u][j], O[u][db]);
            O[u][db] = mfma_16x16x32(vf, pl[u][j], O[u][db]);        // O^T[dim 16 db + 4 g + r][query qi of tile u]
          }
        }
      }
  }
  const float sk = a.sink ? a.sink[h] * 1.44269504088896340736f : -INFINITY;
#pragma unroll
  for (int u = 0; u < LP_QT; ++u) {
    float L = l[u];
    L += __shfl_xor(L, 16, WAVE);
    L += __shfl_xor(L, 32, WAVE);
    const int i = wq + u * 16 + qi;
    if (i >= tile.y) continue;
    const float M = fmaxf(m[u], sk);
    const float f = exp2f(m[u] - M);
    const float inv = f / (L * f + (sk == -INFINITY ? 0.f : exp2f(sk - M)));
    const int t = tile.x + i;
#pragma unroll
    for (int db = 0; db < VB_; ++db) {
      if (EXACT || db < VB) {
        const int col = (h * VB + db) * 16 + 4 * g;
        elt* p = a.frag_tt ? a.out + frag_offset(t, col, a.frag_tt) : a.out + (size_t)t * a.ld_out + col;
        *reinterpret_cast<eltx4*>(p) =
            eltx4{(elt)(O[u][db][0] * inv), (elt)(O[u][db][1] * inv), (elt)(O[u][db][2] * inv), (elt)(O[u][db][3] * inv)};
      }
    }
  }
}

// y[t, h] = alpha * W[h] . x[t, h] per head: W[h] packed [N, K], N % 16 == 0.  A wave owns 16 NI rows x 16 TJ tokens.
struct HeadLinear {
  elt* y;
  long ldy, hy;
  int frag_tt;
  const elt* x;
  long ldx, hx;
  const elt* W;
  int T, K, N;
  float alpha;
};

template <int NI, int TJ>
__device__ __forceinline__ void head_linear(const HeadLinear& a, int bx, int by, int h) {
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int t0 = by * 16 * TJ;
  const int KB = a.K / 32, tiles = a.N / 16, nt0 = (bx * 4 + wave) * NI;
  if (nt0 >= tiles) return;
  const int r16 = lane & 15, g = lane >> 4;
  const elt* wp[NI];
  const elt* xp[TJ];
#pragma unroll
  for (int i = 0; i < NI; ++i) wp[i] = a.W + ((size_t)h * tiles + (nt0 + i < tiles ? nt0 + i : tiles - 1)) * KB * 512 + lane * 8;
#pragma unroll
  for (int j = 0; j < TJ; ++j) {
    const int t = t0 + j * 16 + r16;
    xp[j] = a.x + (t < a.T ? t : a.T - 1) * a.ldx + h * a.hx + g * 8;
  }
  f32x4 acc[NI][TJ];
#pragma unroll
  for (int i = 0; i < NI; ++i)
#pragma unroll
    for (int j = 0; j < TJ; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  constexpr int U = NI * TJ > 4 ? 1 : 4;                             // k-steps requested together
  for (int k0 = 0; k0 < KB; k0 += U) {
    eltx8 w[U][NI], b[U][TJ];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int ks = k0 + u < KB ? k0 + u : k0;                      // past K: a valid address, zeroed
#pragma unroll
      for (int i = 0; i < NI; ++i) w[u][i] = ld8(wp[i] + (size_t)ks * 512);
#pragma unroll
      for (int j = 0; j < TJ; ++j) {
        b[u][j] = ld8(xp[j] + ks * 32);
        if (k0 + u >= KB) b[u][j] = eltx8{0, 0, 0, 0, 0, 0, 0, 0};
      }
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int i = 0; i < NI; ++i)
#pragma unroll
        for (int j = 0; j < TJ; ++j) acc[i][j] = mfma_16x16x32(w[u][i], b[u][j], acc[i][j]);
  }
#pragma unroll
  for (int j = 0; j < TJ; ++j) {
    const int t = t0 + j * 16 + r16;
    if (t >= a.T) continue;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int n = (nt0 + i) * 16 + g * 4;
      if (n >= a.N) continue;
      const f32x4 s = acc[i][j] * a.alpha;
      elt* p = a.frag_tt ? a.y + frag_offset(t, (int)(h * a.hy) + n, a.frag_tt) : a.y + t * a.ldy + h * a.hy + n;
      *reinterpret_cast<eltx4*>(p) = eltx4{(elt)s[0], (elt)s[1], (elt)s[2], (elt)s[3]};
    }
  }
}

template <int NI, int TJ>
__global__ __launch_bounds__(256, 2) void head_linear_kernel(HeadLinear a) {
  head_linear<NI, TJ>(a, blockIdx.x, blockIdx.y, blockIdx.z);
}

// latent_prep and the lifting of the queries (which need nothing of each other) in one launch: T workgroups, then nx * ny * H
template <int TJ>
__global__ __launch_bounds__(256, 2) void latent_query_kernel(LatentPrep p, HeadLinear a, int nx, int ny) {
  __shared__ float red[4];
  int b = blockIdx.x;
  if (b < a.T) return latent_prep(p, b, red);                        // uniform
  b -= a.T;
  const int bx = b % nx, r = b / nx;
  head_linear<1, TJ>(a, bx, r % ny, r / ny);
}

// The splits of (16 tokens, head) added - with the sink's share of the denominator - and taken through W_uv in one launch:
// the merged context vectors meet the matrix cores from LDS.  grid (H, token tiles).
constexpr int LO_SPLITS = 32;
constexpr int LO_WAVES = 8;
constexpr int LO_PRE = 8;          // weight fragments of a wave's first tile that are requested ahead of the merge
__global__ __launch_bounds__(LO_WAVES* WAVE, 2) void latent_out_kernel(LatentAttn a, HeadLinear o) {
  extern __shared__ __align__(16) elt xs[];                          // [RB][64][8]
  __shared__ float fs[LO_SPLITS][16], ls[LO_SPLITS][16];
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int h = blockIdx.x, t0 = blockIdx.y * 16, rd = a.RB * 32, tiles = o.N / 16;
  const size_t n = (size_t)a.T * a.H;
  for (int i = threadIdx.x; i < a.splits * 16; i += LO_WAVES * WAVE) {
    const int t = t0 + (i & 15) < a.T ? t0 + (i & 15) : a.T - 1;
    const float* ml = a.part_ml + 2 * (((size_t)(i >> 4) * a.T + t) * a.H + h);
    fs[i >> 4][i & 15] = ml[0];
    ls[i >> 4][i & 15] = ml[1];
  }
  const elt* wp = o.W + (size_t)h * tiles * a.RB * 512 + lane * 8;
  eltx8 w[LO_PRE];
#pragma unroll
  for (int u = 0; u < LO_PRE; ++u) w[u] = ld8(wp + ((size_t)(wave < tiles ? wave : 0) * a.RB + (u < a.RB ? u : 0)) * 512);
  __syncthreads();
  if (threadIdx.x < 16) {
    const float sk = a.sink ? a.sink[h] : -INFINITY;
    float M = sk;
    for (int s = 0; s < a.splits; ++s) M = fmaxf(M, fs[s][threadIdx.x]);
    float L = sk != -INFINITY ? __expf(sk - M) : 0.f;
    for (int s = 0; s < a.splits; ++s) {
      const float m = fs[s][threadIdx.x], f = m == -INFINITY ? 0.f : __expf(m - M);
      fs[s][threadIdx.x] = f;
      L += ls[s][threadIdx.x] * f;
    }
    const float inv = L > 0.f ? 1.f / L : 0.f;
    for (int s = 0; s < a.splits; ++s) fs[s][threadIdx.x] *= inv;
  }
  // the splits are added as they come: four splits of a thread's eight values are in flight at a time
  for (int i0 = 0; i0 < a.RB * 64; i0 += LO_WAVES * WAVE) {
    const int i = i0 + threadIdx.x, ic = i < a.RB * 64 ? i : 0, tk = ic & 15, t = t0 + tk < a.T ? t0 + tk : a.T - 1;
    const float* p = a.part_o + ((size_t)t * a.H + h) * rd + (ic >> 6) * 32 + ((ic >> 4) & 3) * 8;
    f32x4 lo = f32x4{0.f, 0.f, 0.f, 0.f}, hi = lo;
    for (int s0 = 0; s0 < a.splits; s0 += 4) {
      f32x4 v[4][2];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const float* ps = p + (size_t)(s0 + u < a.splits ? s0 + u : s0) * n * rd;
        v[u][0] = *reinterpret_cast<const f32x4*>(ps);
        v[u][1] = *reinterpret_cast<const f32x4*>(ps + 4);
      }
      if (i0 == 0 && s0 == 0) __syncthreads();                       // the factors
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const float f = s0 + u < a.splits ? fs[s0 + u][tk] : 0.f;
        lo += v[u][0] * f;
        hi += v[u][1] * f;
      }
    }
    if (i < a.RB * 64)
      st8(xs + i * 8, eltx8{(elt)lo[0], (elt)lo[1], (elt)lo[2], (elt)lo[3], (elt)hi[0], (elt)hi[1], (elt)hi[2], (elt)hi[3]});
  }
  __syncthreads();
  const int r16 = lane & 15, g = lane >> 4, t = t0 + r16;
  for (int nt = wave; nt < tiles; nt += LO_WAVES) {
    f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < a.RB; k0 += LO_PRE) {
      if (nt != wave || k0 > 0) {                                    // uniform
#pragma unroll
        for (int u = 0; u < LO_PRE; ++u) w[u] = ld8(wp + ((size_t)nt * a.RB + (k0 + u < a.RB ? k0 + u : k0)) * 512);
      }
#pragma unroll
      for (int u = 0; u < LO_PRE; ++u)
        if (k0 + u < a.RB) acc = mfma_16x16x32(w[u], ld8(xs + ((k0 + u) * 64 + lane) * 8), acc);   // uniform
    }
    if (t >= a.T) continue;
    const int c = nt * 16 + g * 4;
    elt* p = o.frag_tt ? o.y + frag_offset(t, (int)(h * o.hy) + c, o.frag_tt) : o.y + t * o.ldy + h * o.hy + c;
    *reinterpret_cast<eltx4*>(p) = eltx4{(elt)acc[0], (elt)acc[1], (elt)acc[2], (elt)acc[3]};
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
  const int kvh = h / a.gs;                       // one key/value head unless tied
  const float slope = a.slopes ? a.slopes[h] : 0.f;
  float m = a.sink ? a.sink[h] : -INFINITY, l = a.sink ? 1.f : 0.f, o[LA_DPT] = {};
  for (int j0 = 0; j0 < ctx; j0 += LA_KEYS) {
    __syncthreads();
    if (threadIdx.x < LA_KEYS / PAGE) {
      const int pg = j0 / PAGE + threadIdx.x;
      const int page = pg * PAGE < ctx ? bt[pg] : -1;
      pgs[threadIdx.x] = page >= 0 && page < a.n_pages ? page * a.G + kvh : -1;
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
      if (a.key_scale) s *= a.key_scale[(size_t)page * PAGE + j % PAGE];
      if (a.slopes) s = fmaf(-slope, (float)(ctx - 1 - j), s);
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
template <int NRB, int NW, bool TIED = false>
int launch_latent_attn(const LatentAttn& a, hipStream_t s) {
  const int kr = a.NB - a.RB;
  const size_t lds = (size_t)(a.chunks * NRB + (TIED ? 0 : kr > 2 ? kr : 2)) * 1024 + (size_t)NW * 16 * 68 * sizeof(float);
  static const hipError_t configured =               // the attribute is per kernel, set once per process, by one thread
      hipFuncSetAttribute((const void*)latent_attn_kernel<NRB, NW, TIED>, hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);
  if (configured != hipSuccess || lds > 96 * 1024)
    return mlora_set_error(MLORA_ERR_UNSUPPORTED, "latent_attn: cannot reserve %zu bytes of LDS", lds);
  const long outer = ((long)a.T * a.splits + 7) / 8 * 8;
  if (outer * a.n_inner > 0x7fffffffL) return mlora_set_error(MLORA_ERR_UNSUPPORTED, "latent_attn: T=%d is too many tokens", a.T);
  hipLaunchKernelGGL((latent_attn_kernel<NRB, NW, TIED>), dim3((unsigned)(outer * a.n_inner)), dim3(NW * WAVE), lds, s, a);
  return MLORA_OK;
}
#endif

// ---------------------------------------------------------------------------------------------
// Tied attention
// ---------------------------------------------------------------------------------------------
struct TiedPrep {
  const float* y;           // [T, ld]: projections without their biases, the H query heads' and then the G key/value heads' D columns each
  int ld;
  const float* bias;        // [(H + G) D]
  const float* q_norm;      // [D]: the queries' norm weight (times that of the keys, where the keys go without)
  float eps, temp_coef, temp_every;
  elt* q;                   // [T, H, RB * 32]
  elt* cache;
  float* key_scale;
  const int32_t* block_table;
  int max_blocks, n_pages, n_seq;
  const int32_t* tok_seq;
  const int32_t* tok_pos;
  int T, H, G, D, RB;
};

constexpr int TP_MAX_D = 512;
// LN lanes per (token, head), eight columns each: adds the bias; a query is normed and takes its temperature, a value goes to the
// token's page slot with the reciprocal of its root mean square.  VEC: whole eights of columns, 16-byte aligned.
template <int LN, bool VEC>
__global__ __launch_bounds__(256) void tied_prep_kernel(TiedPrep a) {
  const int d = (threadIdx.x % LN) * 8, hh = blockIdx.y * (256 / LN) + threadIdx.x / LN, t = blockIdx.x;
  if (hh >= a.H + a.G) return;                                       // whole groups of LN lanes; no barrier below
  const int seq = a.tok_seq[t], pos = a.tok_pos[t], Dp = a.RB * 32;
  const float* yp = a.y + (size_t)t * a.ld + hh * a.D + d;
  const float* bp = a.bias + hh * a.D + d;
  f32x4 v[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}}, w[2] = {v[0], v[0]};
  if constexpr (VEC) {
    if (d < a.D) {
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        v[i] = *reinterpret_cast<const f32x4*>(yp + 4 * i) + *reinterpret_cast<const f32x4*>(bp + 4 * i);
        w[i] = *reinterpret_cast<const f32x4*>(a.q_norm + d + 4 * i);
      }
    }
  } else {
#pragma unroll
    for (int e = 0; e < 8; ++e)
      if (d + e < a.D) {
        v[e >> 2][e & 3] = yp[e] + bp[e];
        w[e >> 2][e & 3] = a.q_norm[d + e];
      }
  }
  float ss = 0.f;
#pragma unroll
  for (int e = 0; e < 8; ++e) ss = fmaf(v[e >> 2][e & 3], v[e >> 2][e & 3], ss);
#pragma unroll
  for (int o = LN / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, WAVE);
  const float inv = 1.f / sqrtf(ss / (float)a.D + a.eps);
  eltx8 o;
  if (hh < a.H) {
    float f = inv;
    if (a.temp_every > 0.f) f *= fmaf(a.temp_coef, logf(floorf((float)(pos + 1) / a.temp_every) + 1.f), 1.f);
#pragma unroll
    for (int e = 0; e < 8; ++e) o[e] = (elt)(v[e >> 2][e & 3] * f * w[e >> 2][e & 3]);
    if (d < Dp) st8(a.q + ((size_t)t * a.H + hh) * Dp + d, o);
    return;
  }
  if (seq < 0 || seq >= a.n_seq || pos < 0 || pos / PAGE >= a.max_blocks) return;
  const int page = a.block_table[(size_t)seq * a.max_blocks + pos / PAGE];
  if (page < 0 || page >= a.n_pages) return;
  const int pg = page * a.G + hh - a.H;
#pragma unroll
  for (int e = 0; e < 8; ++e) o[e] = (elt)v[e >> 2][e & 3];
  if (d < Dp) st8(a.cache + latent_offset(pg, a.RB, pos % PAGE, d), o);
  if (d == 0) a.key_scale[(size_t)pg * PAGE + pos % PAGE] = inv;
}

template <int LN>
void launch_tied_prep(const TiedPrep& a, hipStream_t s) {
  const dim3 grid(a.T, ceil_div(a.H + a.G, 256 / LN));
  if (a.D % 8 == 0 && a.ld % 4 == 0 && (((uintptr_t)a.y | (uintptr_t)a.bias | (uintptr_t)a.q_norm) & 15) == 0)
    hipLaunchKernelGGL((tied_prep_kernel<LN, true>), grid, dim3(256), 0, s, a);
  else
    hipLaunchKernelGGL((tied_prep_kernel<LN, false>), grid, dim3(256), 0, s, a);
}

#ifndef MLORA_ELT_F32
// The keys (normed, without the weight, which the queries carry) and the transposed values of whole contexts in the scratch
// layouts of the prompt form, K [G, pages, RB, 512] and V [G, pages / 2, 2 RB, 512]: one workgroup per (pair of pages, key/value head).
__global__ __launch_bounds__(256) void tied_expand_kernel(elt* __restrict__ k, elt* __restrict__ v, const elt* __restrict__ cache,
                                                          const float* __restrict__ key_scale, const int32_t* __restrict__ phys, int pages,
                                                          int n_pages, int G, int RB) {
  const int pp = blockIdx.x, kvh = blockIdx.y;
  int pg[2];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    pg[j] = phys[2 * pp + j];
    pg[j] = pg[j] >= 0 && pg[j] < n_pages ? pg[j] * G + kvh : -1;
  }
  for (int i = threadIdx.x; i < 2 * RB * 64; i += 256) {             // keys: a page's fragments, each token's row scaled
    const int j = i / (RB * 64), o = i - j * (RB * 64);
    eltx8 x = eltx8{0, 0, 0, 0, 0, 0, 0, 0};
    if (pg[j] >= 0) {
      const float s = key_scale[(size_t)pg[j] * PAGE + (o & 15)];
      x = ld8(cache + (size_t)pg[j] * RB * 512 + o * 8);
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] = (elt)((float)x[e] * s);
    }
    st8(k + (((size_t)kvh * pages + 2 * pp + j) * RB * 64 + o) * 8, x);
  }
  for (int i = threadIdx.x; i < 2 * RB * 64; i += 256) {             // values: 16 dims x 32 tokens per fragment
    const int db = i >> 6, l = i & 63, d = db * 16 + (l & 15), g = l >> 4;
    eltx8 x = eltx8{0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
    for (int j = 0; j < 2; ++j)
      if (pg[j] >= 0) {
#pragma unroll
        for (int r = 0; r < 4; ++r) x[j * 4 + r] = cache[latent_offset(pg[j], RB, 4 * g + r, d)];
      }
    st8(v + (((size_t)kvh * (pages / 2) + pp) * 2 * RB * 64 + i) * 8, x);
  }
}
#endif

}  // namespace

// lift [H * RB * 32, lift_k] packed (or NULL): the unrotated query parts (columns 0.. of qkv, lift_k per head) lifted into q
extern "C" int mlora_latent_prep(void* q, int q_ld, int q_off, void* cache, const void* qkv, int ld, int off_rot, int off_c, int off_kr, float gain, const void* c_norm,
                                 float eps, const int32_t* block_table, int max_blocks, const int32_t* tok_seq, const int32_t* tok_pos,
                                 const float* rope_cos, const float* rope_sin, int max_pos, int T, int H, int R, int rot, int n_pages, int n_seq,
                                 const void* lift, int lift_k, void* stream) {
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
  a.q_ld = q_ld; a.q_off = q_off;
  MLORA_CHECK(q_off >= 0 && q_off % 2 == 0 && q_ld % 2 == 0 && q_off + (a.NB - a.RB) * 32 <= q_ld, MLORA_ERR_INVALID,
              "latent_prep: query rows of %d with the rotated part at %d", q_ld, q_off);
#ifndef MLORA_ELT_F32
  if (lift) {
    MLORA_CHECK(lift_k > 0 && lift_k % 32 == 0 && H * lift_k <= ld && ld % 8 == 0 && q_off == a.RB * 32 && q_ld % 4 == 0, MLORA_ERR_UNSUPPORTED,
                "latent_prep: lifting needs query parts of whole 32 columns ahead of the rest (lift_k=%d ld=%d)", lift_k, ld);
    HeadLinear l;
    l.y = (elt*)q; l.ldy = (long)H * q_ld; l.hy = q_ld; l.frag_tt = 0;
    l.x = (const elt*)qkv; l.ldx = ld; l.hx = lift_k; l.W = (const elt*)lift; l.T = T; l.K = lift_k; l.N = a.RB * 32; l.alpha = 1.f;
    const int nx = ceil_div(l.N, 64), tj = T <= 16 ? 1 : T <= 256 ? 2 : 4, ny = ceil_div(T, 16 * tj);
    const long blocks = T + (long)nx * ny * H;
    MLORA_CHECK(blocks <= 0x7fffffffL, MLORA_ERR_UNSUPPORTED, "latent_prep: T=%d is too many tokens", T);
    hipStream_t s = (hipStream_t)stream;
    if (tj == 1) hipLaunchKernelGGL(latent_query_kernel<1>, dim3((unsigned)blocks), dim3(256), 0, s, a, l, nx, ny);
    else if (tj == 2) hipLaunchKernelGGL(latent_query_kernel<2>, dim3((unsigned)blocks), dim3(256), 0, s, a, l, nx, ny);
    else hipLaunchKernelGGL(latent_query_kernel<4>, dim3((unsigned)blocks), dim3(256), 0, s, a, l, nx, ny);
    return mlora_launch_status("latent_prep");
  }
#else
  MLORA_CHECK(!lift, MLORA_ERR_UNSUPPORTED, "latent_prep: the fp32 library lifts queries with mlora_head_linear");
  (void)lift_k;
#endif
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
  int s = (int)(256 / wgs);                                       // a workgroup per compute unit ...
  const int by_ctx = max_ctx / (8 * PAGE);                        // ... of at least one page per wave
  if (s > by_ctx) s = by_ctx;
  if (s > 32) s = 32;
  return s < 1 ? 1 : s;
#endif
}

extern "C" size_t mlora_latent_attn_workspace_bytes(int T, int H, int R, int splits) {
  if (T <= 0 || H <= 0 || R <= 0 || splits <= 1) return 0;
  return (size_t)splits * T * H * ((size_t)ceil_div(R, 32) * 32 + 2) * sizeof(float);
}

// o: a HeadLinear that takes the merged context vectors (nullptr: they go to `out`)
static int latent_attn_impl(void* out, const void* q, const void* cache, const int32_t* block_table, int max_blocks, const int32_t* tok_seq,
                            const int32_t* tok_pos, const float* sink, float scale, int T, int H, int R, int rot, int n_pages, int n_seq,
                            int splits, void* workspace, size_t workspace_bytes, const void* o, void* stream) {
  MLORA_CHECK(T >= 0 && H > 0 && H <= 65535 && R > 0 && rot > 0 && max_blocks > 0 && n_pages > 0 && n_seq > 0 && splits >= 1, MLORA_ERR_INVALID,
              "latent_attn: bad shape T=%d H=%d R=%d rot=%d", T, H, R, rot);
  if (T == 0) return MLORA_OK;
  LatentAttn a = {};
  a.G = 1; a.gs = H;
  a.out = (elt*)out; a.q = (const elt*)q; a.cache = (const elt*)cache; a.block_table = block_table; a.max_blocks = max_blocks;
  a.n_pages = n_pages; a.n_seq = n_seq; a.tok_seq = tok_seq; a.tok_pos = tok_pos; a.sink = sink; a.scale = scale;
  a.T = T; a.H = H; a.RB = ceil_div(R, 32); a.NB = a.RB + ceil_div(rot, 32); a.splits = splits;
  a.part_o = a.part_ml = nullptr; a.n_inner = a.chunks = 1;
  hipStream_t s = (hipStream_t)stream;
#ifdef MLORA_ELT_F32
  (void)o; (void)workspace; (void)workspace_bytes;
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
  if (nrb == 2) e = launch_latent_attn<2, 8>(a, s);
  else if (nrb == 4) e = launch_latent_attn<4, 8>(a, s);
  else if (nrb == 8) e = launch_latent_attn<8, 8>(a, s);
  else e = launch_latent_attn<16, 8>(a, s);
  if (e) return e;
  if (splits > 1) {
    MLORA_CHECK((long)T * H <= 0x7fffffffL, MLORA_ERR_UNSUPPORTED, "latent_attn: T=%d is too many tokens", T);
    if (o) hipLaunchKernelGGL(latent_out_kernel, dim3(H, ceil_div(T, 16)), dim3(LO_WAVES * WAVE), (size_t)a.RB * 1024, s, a, *(const HeadLinear*)o);
    else hipLaunchKernelGGL(latent_merge_kernel, dim3(T * H), dim3(128), 0, s, a);
  }
#endif
  return mlora_launch_status("latent_attn");
}

extern "C" int mlora_latent_attn(void* out, const void* q, const void* cache, const int32_t* block_table, int max_blocks, const int32_t* tok_seq,
                                 const int32_t* tok_pos, const float* sink, float scale, int T, int H, int R, int rot, int n_pages, int n_seq,
                                 int splits, void* workspace, size_t workspace_bytes, void* stream) {
  MLORA_CHECK(out && q && cache && block_table && tok_seq && tok_pos, MLORA_ERR_INVALID, "latent_attn: null pointer");
  return latent_attn_impl(out, q, cache, block_table, max_blocks, tok_seq, tok_pos, sink, scale, T, H, R, rot, n_pages, n_seq, splits, workspace,
                          workspace_bytes, nullptr, stream);
}

#ifndef MLORA_ELT_F32
extern "C" int mlora_latent_attn_out(void* y, int y_layout, long ldy, const void* uv, int vp, const void* q, const void* cache,
                                     const int32_t* block_table, int max_blocks, const int32_t* tok_seq, const int32_t* tok_pos, const float* sink,
                                     float scale, int T, int H, int R, int rot, int n_pages, int n_seq, int splits, void* workspace,
                                     size_t workspace_bytes, void* stream) {
  MLORA_CHECK(y && uv && q && cache && block_table && tok_seq && tok_pos, MLORA_ERR_INVALID, "latent_attn_out: null pointer");
  MLORA_CHECK(splits > 1 && splits <= LO_SPLITS && vp > 0 && vp % 32 == 0 && (y_layout == MLORA_FRAG || ldy % 4 == 0) && ceil_div(T, 16) <= 65535 &&
                  R <= 1536,
              MLORA_ERR_UNSUPPORTED, "latent_attn_out: need 2..%d splits, vp %% 32 == 0 (splits=%d vp=%d R=%d)", LO_SPLITS, splits, vp, R);
  HeadLinear o = {};
  o.y = (elt*)y; o.ldy = ldy; o.hy = vp; o.frag_tt = y_layout == MLORA_FRAG ? mlora_frag_tiles(T) : 0; o.W = (const elt*)uv; o.T = T; o.N = vp;
  return latent_attn_impl(nullptr, q, cache, block_table, max_blocks, tok_seq, tok_pos, sink, scale, T, H, R, rot, n_pages, n_seq, splits, workspace,
                          workspace_bytes, &o, stream);
}
#endif

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
  HeadLinear a;
  a.y = (elt*)y; a.ldy = ldy; a.hy = head_y; a.frag_tt = tt; a.x = (const elt*)x; a.ldx = ldx; a.hx = head_x; a.W = (const elt*)W;
  a.T = T; a.K = K; a.N = N; a.alpha = alpha;
#define MLORA_HL(NI, TJ) \
  hipLaunchKernelGGL((head_linear_kernel<NI, TJ>), dim3(ceil_div(N, 64 * NI), ceil_div(T, 16 * TJ), heads), dim3(256), 0, s, a)
  if (T <= 16) MLORA_HL(1, 1);
  else if (T <= 256) MLORA_HL(1, 2);
  else MLORA_HL(4, 4);
#undef MLORA_HL
  return mlora_launch_status("head_linear");
}
#endif

#ifndef MLORA_ELT_F32
template <int KB, int VB, bool EXACT, bool TIED = false>
static int launch_latent_prefill(const LatentPrefill& a, int n_tiles, hipStream_t s) {
  constexpr size_t cap = (size_t)2 * (4 * KB + 2 * VB) * 512 * sizeof(elt);
  static const hipError_t configured =               // the attribute is per kernel, set once per process, by one thread
      hipFuncSetAttribute((const void*)latent_prefill_kernel<KB, VB, EXACT, TIED>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)cap);
  if (configured != hipSuccess) return mlora_set_error(MLORA_ERR_LAUNCH, "latent_prefill: cannot reserve %zu bytes of LDS", cap);
  const size_t lds = (size_t)2 * (4 * (a.KN + a.KR) + 2 * a.VB) * 512 * sizeof(elt);
  hipLaunchKernelGGL((latent_prefill_kernel<KB, VB, EXACT, TIED>), dim3(a.H, n_tiles), dim3(LP_WAVES * WAVE), lds, s, a);
  return MLORA_OK;
}

extern "C" int mlora_latent_prefill_tile_tokens(void) { return LP_TOK; }

extern "C" int mlora_latent_prefill_served(int dim, int rot, int vdim) {
  return dim > 0 && rot > 0 && vdim > 0 && ceil_div(dim, 32) + ceil_div(rot, 32) <= 6 && ceil_div(vdim, 32) <= 4;
}

// elements of scratch memory for `pages` scratch pages
extern "C" size_t mlora_latent_prefill_scratch_elems(int pages, int H, int dim, int rot, int vdim) {
  if (pages <= 0 || H <= 0) return 0;
  return (size_t)pages * 512 * ((size_t)H * (ceil_div(dim, 32) + ceil_div(vdim, 32)) + ceil_div(rot, 32));
}

extern "C" int mlora_latent_prefill(void* out, int out_layout, int ld_out, const void* q, int ld_q, const void* q_rot, const void* cache,
                                    const int32_t* phys, int pages, const int32_t* tiles, int n_tiles, const void* uk, const void* uv,
                                    const float* sink, float scale, int T, int H, int R, int dim, int rot, int vdim, int n_pages, void* scratch,
                                    size_t scratch_elems, void* stream) {
  MLORA_CHECK(out && q && q_rot && cache && phys && tiles && uk && uv && scratch, MLORA_ERR_INVALID, "latent_prefill: null pointer");
  MLORA_CHECK(mlora_latent_prefill_served(dim, rot, vdim) && H > 0 && H <= 65535 && R > 0 && n_pages > 0, MLORA_ERR_UNSUPPORTED,
              "latent_prefill: dim=%d rot=%d vdim=%d not served", dim, rot, vdim);
  MLORA_CHECK(pages > 0 && pages % 4 == 0 && pages / 4 <= 65535 && n_tiles > 0 && n_tiles <= 65535 && T > 0 && ld_q % 8 == 0 &&
                  (((uintptr_t)q | (uintptr_t)q_rot | (uintptr_t)scratch | (uintptr_t)tiles) & 15) == 0,
              MLORA_ERR_UNSUPPORTED, "latent_prefill: pages=%d must be a multiple of 4, operands aligned", pages);
  MLORA_CHECK((long)H * (ceil_div(dim, 32) + ceil_div(vdim, 32)) * ceil_div(R, 32) * 1024 < (1L << 31), MLORA_ERR_UNSUPPORTED,
              "latent_prefill: weights too large (H=%d R=%d)", H, R);
  MLORA_CHECK(scratch_elems >= mlora_latent_prefill_scratch_elems(pages, H, dim, rot, vdim), MLORA_ERR_WORKSPACE, "latent_prefill: scratch too small");
  LatentExpand e;
  e.KN = ceil_div(dim, 32); e.KR = ceil_div(rot, 32); e.VB = ceil_div(vdim, 32) * 2; e.RB = ceil_div(R, 32);
  e.H = H; e.pages = pages; e.n_pages = n_pages;
  e.k = (elt*)scratch;
  e.v = e.k + (size_t)H * pages * e.KN * 512;
  e.r = e.v + (size_t)H * (pages / 2) * e.VB * 512;
  e.cache = (const elt*)cache; e.phys = phys; e.uk = (const elt*)uk; e.uv = (const elt*)uv;
  e.kb_blocks = ceil_div(H * e.KN * 2, 4 * LE_ROWS);
  e.vb_blocks = ceil_div(H * e.VB, 4 * LE_ROWS);
  hipStream_t s = (hipStream_t)stream;
  hipLaunchKernelGGL(latent_expand_kernel, dim3((e.kb_blocks + e.vb_blocks + 1 + 7) / 8 * 8, ceil_div(pages, 8)), dim3(512), 0, s, e);   // whole eights: a weight row stays on one XCD
  LatentPrefill a = {};
  a.out = (elt*)out; a.frag_tt = out_layout == MLORA_FRAG ? mlora_frag_tiles(T) : 0; a.ld_out = ld_out;
  a.q = (const elt*)q; a.ld_q = ld_q; a.qr = (const elt*)q_rot; a.k = e.k; a.v = e.v; a.r = e.r; a.tiles = (const int4*)tiles;
  a.sink = sink; a.scale = scale; a.H = H; a.pages = pages; a.KN = e.KN; a.KR = e.KR; a.VB = e.VB;
  const int KB = e.KN + e.KR;
  int rc;
  if (KB == 6 && e.VB == 8) rc = launch_latent_prefill<6, 8, true>(a, n_tiles, s);
  else if (KB <= 3 && e.VB <= 4) rc = launch_latent_prefill<3, 4, false>(a, n_tiles, s);
  else rc = launch_latent_prefill<6, 8, false>(a, n_tiles, s);
  return rc ? rc : mlora_launch_status("latent_prefill");
}
#endif

// ---------------------------------------------------------------------------------------------
// Tied attention
// ---------------------------------------------------------------------------------------------
extern "C" int mlora_tied_prep(void* q, void* cache, float* key_scale, const float* y, int ld, const float* bias, const float* q_norm, float eps,
                               float temp_coef, float temp_every, const int32_t* block_table, int max_blocks, const int32_t* tok_seq,
                               const int32_t* tok_pos, int T, int H, int G, int D, int n_pages, int n_seq, void* stream) {
  MLORA_CHECK(q && cache && key_scale && y && bias && q_norm && block_table && tok_seq && tok_pos, MLORA_ERR_INVALID, "tied_prep: null pointer");
  MLORA_CHECK(T >= 0 && H > 0 && G > 0 && H % G == 0 && D > 0 && D <= TP_MAX_D && ld >= (H + G) * D && max_blocks > 0 && n_pages > 0 && n_seq > 0 &&
                  (long)n_pages * G <= 0x7fffffffL && ceil_div(H + G, 4) <= 65535,
              MLORA_ERR_UNSUPPORTED, "tied_prep: need whole groups of heads of at most %d columns (T=%d H=%d G=%d D=%d)", TP_MAX_D, T, H, G, D);
  if (T == 0) return MLORA_OK;
  TiedPrep a;
  a.y = y; a.ld = ld; a.bias = bias; a.q_norm = q_norm; a.eps = eps; a.temp_coef = temp_coef; a.temp_every = temp_every; a.q = (elt*)q;
  a.cache = (elt*)cache; a.key_scale = key_scale; a.block_table = block_table; a.max_blocks = max_blocks; a.n_pages = n_pages; a.n_seq = n_seq;
  a.tok_seq = tok_seq; a.tok_pos = tok_pos; a.T = T; a.H = H; a.G = G; a.D = D; a.RB = ceil_div(D, 32);
  hipStream_t s = (hipStream_t)stream;
  if (D <= 32) launch_tied_prep<4>(a, s);
  else if (D <= 64) launch_tied_prep<8>(a, s);
  else if (D <= 128) launch_tied_prep<16>(a, s);
  else if (D <= 256) launch_tied_prep<32>(a, s);
  else launch_tied_prep<64>(a, s);
  return mlora_launch_status("tied_prep");
}

extern "C" int mlora_tied_attn_splits(int T, int H, int G, int max_ctx) {
#ifdef MLORA_ELT_F32
  return 1;
#else
  if (T <= 0 || G <= 0 || H < G || max_ctx <= 0) return 1;
  const long wgs = (long)T * G * ceil_div(H / G, 16);
  int s = (int)(512 / wgs);                                       // two workgroups per compute unit ...
  const int by_ctx = max_ctx / (8 * PAGE);                        // ... of at least one page per wave
  if (s > by_ctx) s = by_ctx;
  if (s > 32) s = 32;
  return s < 1 ? 1 : s;
#endif
}

extern "C" int mlora_tied_attn(void* out, int out_layout, const void* q, const void* cache, const float* key_scale, const int32_t* block_table,
                               int max_blocks, const int32_t* tok_seq, const int32_t* tok_pos, const float* slopes, float scale, int T, int H, int G,
                               int D, int n_pages, int n_seq, int splits, void* workspace, size_t workspace_bytes, void* stream) {
  MLORA_CHECK(out && q && cache && key_scale && slopes && block_table && tok_seq && tok_pos, MLORA_ERR_INVALID, "tied_attn: null pointer");
  MLORA_CHECK(T >= 0 && H > 0 && H <= 65535 && G > 0 && H % G == 0 && D > 0 && D <= 512 && max_blocks > 0 && n_pages > 0 && n_seq > 0 && splits >= 1 &&
                  (long)n_pages * G <= 0x7fffffffL && (out_layout == MLORA_ROWMAJOR || sizeof(elt) == 2),
              MLORA_ERR_UNSUPPORTED, "tied_attn: bad shape T=%d H=%d G=%d D=%d", T, H, G, D);
  if (T == 0) return MLORA_OK;
  LatentAttn a = {};
  a.out = (elt*)out; a.q = (const elt*)q; a.cache = (const elt*)cache; a.block_table = block_table; a.max_blocks = max_blocks;
  a.n_pages = n_pages; a.n_seq = n_seq; a.tok_seq = tok_seq; a.tok_pos = tok_pos; a.scale = scale; a.T = T; a.H = H;
  a.RB = a.NB = ceil_div(D, 32); a.splits = splits; a.key_scale = key_scale; a.slopes = slopes; a.G = G; a.gs = H / G; a.gt = ceil_div(H / G, 16); a.D = D;
  a.frag_tt = out_layout == MLORA_FRAG ? mlora_frag_tiles(T) : 0; a.chunks = 1;
  hipStream_t s = (hipStream_t)stream;
#ifdef MLORA_ELT_F32
  (void)workspace; (void)workspace_bytes;
  MLORA_CHECK(splits == 1, MLORA_ERR_UNSUPPORTED, "tied_attn: splits=%d not served in fp32", splits);
  hipLaunchKernelGGL(latent_attn_f32_kernel, dim3(T, H, ceil_div(a.RB * 32, 256 * LA_DPT)), dim3(256), a.NB * 128, s, a);
#else
  if (splits > 1) {
    MLORA_CHECK(workspace && workspace_bytes >= mlora_latent_attn_workspace_bytes(T, H, D, splits), MLORA_ERR_WORKSPACE,
                "tied_attn: workspace of %zu bytes needed", mlora_latent_attn_workspace_bytes(T, H, D, splits));
    MLORA_CHECK((long)T * H <= 0x7fffffffL, MLORA_ERR_UNSUPPORTED, "tied_attn: T=%d is too many tokens", T);
    a.part_o = (float*)workspace;
    a.part_ml = a.part_o + (size_t)splits * T * H * a.RB * 32;
  }
  a.n_inner = G * a.gt;
  int e;
  if (a.RB <= 2) e = launch_latent_attn<2, 8, true>(a, s);
  else if (a.RB <= 4) e = launch_latent_attn<4, 8, true>(a, s);
  else if (a.RB <= 8) e = launch_latent_attn<8, 8, true>(a, s);
  else e = launch_latent_attn<16, 8, true>(a, s);
  if (e) return e;
  if (splits > 1) hipLaunchKernelGGL(latent_merge_kernel, dim3(T * H), dim3(128), 0, s, a);
#endif
  return mlora_launch_status("tied_attn");
}

#ifndef MLORA_ELT_F32
extern "C" int mlora_tied_prefill_served(int D) { return D > 0 && D <= 128; }

extern "C" size_t mlora_tied_prefill_scratch_elems(int pages, int G, int D) {
  if (pages <= 0 || G <= 0 || D <= 0) return 0;
  return (size_t)pages * G * ceil_div(D, 32) * 1024;
}

extern "C" int mlora_tied_prefill(void* out, int out_layout, int ld_out, const void* q, const void* cache, const float* key_scale, const int32_t* phys,
                                  int pages, const int32_t* tiles, int n_tiles, const float* slopes, float scale, int T, int H, int G, int D,
                                  int n_pages, void* scratch, size_t scratch_elems, void* stream) {
  MLORA_CHECK(out && q && cache && key_scale && phys && tiles && slopes && scratch, MLORA_ERR_INVALID, "tied_prefill: null pointer");
  MLORA_CHECK(mlora_tied_prefill_served(D) && H > 0 && H <= 65535 && G > 0 && H % G == 0 && n_pages > 0 && (long)n_pages * G <= 0x7fffffffL,
              MLORA_ERR_UNSUPPORTED, "tied_prefill: H=%d G=%d D=%d not served", H, G, D);
  MLORA_CHECK(pages > 0 && pages % 4 == 0 && n_tiles > 0 && n_tiles <= 65535 && T > 0 && (((uintptr_t)q | (uintptr_t)scratch | (uintptr_t)tiles) & 15) == 0,
              MLORA_ERR_UNSUPPORTED, "tied_prefill: pages=%d must be a multiple of 4, operands aligned", pages);
  MLORA_CHECK(scratch_elems >= mlora_tied_prefill_scratch_elems(pages, G, D), MLORA_ERR_WORKSPACE, "tied_prefill: scratch too small");
  hipStream_t s = (hipStream_t)stream;
  LatentPrefill a = {};
  a.KN = ceil_div(D, 32); a.KR = 0; a.VB = 2 * a.KN; a.H = H; a.pages = pages; a.gs = H / G; a.D = D;
  elt* k = (elt*)scratch;
  elt* v = k + (size_t)G * pages * a.KN * 512;
  hipLaunchKernelGGL(tied_expand_kernel, dim3(pages / 2, G), dim3(256), 0, s, k, v, (const elt*)cache, key_scale, phys, pages, n_pages, G, a.KN);
  a.out = (elt*)out; a.frag_tt = out_layout == MLORA_FRAG ? mlora_frag_tiles(T) : 0; a.ld_out = ld_out;
  a.q = (const elt*)q; a.ld_q = H * a.KN * 32; a.k = k; a.v = v; a.r = k; a.tiles = (const int4*)tiles; a.scale = scale; a.slopes = slopes;
  int rc;
  if (a.KN == 4) rc = launch_latent_prefill<4, 8, true, true>(a, n_tiles, s);
  else if (a.KN == 2) rc = launch_latent_prefill<2, 4, true, true>(a, n_tiles, s);
  else rc = launch_latent_prefill<4, 8, false, true>(a, n_tiles, s);
  return rc ? rc : mlora_launch_status("tied_prefill");
}
#endif
