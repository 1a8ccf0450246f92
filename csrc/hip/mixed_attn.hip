// Causal attention over the paged cache whose softmax WEIGHTS are mixed over the heads:
//
//   s_g(i, j)  = (q_g(i) . k_c(g)(j)) * scale,   j <= i             c(g) = g / (H / G): grouped key/value heads
//   p_g(i, j)  = exp(s_g(i, j)) / sum_j' exp(s_g(i, j'))
//   w_h(i, j)  = sum_g M[h, g] p_g(i, j)                            M [H, H]
//   o_h(i)     = out_scale * sum_j w_h(i, j) v_c(h)(j)
//
// The weights are mixed AFTER the normalisation, so a head's output needs every head's denominator before the first value
// is weighted: two passes over the keys. The first leaves the pair (maximum, sum of exponentials) of every (query, head)
// and key range (`part_ml`), the second forms normalised weights, mixes them and accumulates w.v. Key ranges may be split
// over workgroups (decoding); the second pass merges all splits' pairs before it starts, so its partial results only have
// to be added up.
//
// Scores, weights and sums run in fp32 whatever the storage type T (bf16 / fp32) of q, the caches and the output.
// Queries of row b are the LAST cu_q[b+1] - cu_q[b] positions of its context of ctx_len[b] tokens.
//
// The any-size kernel serves both passes of prompt portions and decoding (with a split key range); bf16 rows of the common
// sizes take the matrix-core kernels further down.
//
// Cache layout: K [pages, G, 32, D], V [pages, G, V, 32] (a channel's 32 tokens side by side).
#include "common.hpp"

namespace {

constexpr int PAGE = 32;
constexpr float LOG2E = 1.4426950408889634f;

template <typename T> DEVINL float ldf(const T* p, size_t i);
template <> DEVINL float ldf<bf16_t>(const bf16_t* p, size_t i) { return bf2f(p[i]); }
template <> DEVINL float ldf<float>(const float* p, size_t i) { return p[i]; }
template <typename T> DEVINL void stf(T* p, size_t i, float v);
template <> DEVINL void stf<bf16_t>(bf16_t* p, size_t i, float v) { p[i] = f2bf(v); }
template <> DEVINL void stf<float>(float* p, size_t i, float v) { p[i] = v; }

// ------------------------------------------------------------------------------------------------------------------
// Any sizes. One workgroup owns all heads of a tile of BQ queries and one share of the keys.
struct MixShape {
  int H, G, D, V, BQ;
  // LDS in floats of the pass that ends in outputs (the other one needs less)
  __host__ __device__ size_t floats() const {
    const size_t R = (size_t)H * BQ;
    return R * D + R * V + 2 * R * PAGE + (size_t)PAGE * (D + 1) + (size_t)V * (PAGE + 1) + 2 * R + (size_t)H * H;
  }
};

// raw scores of one key/value head's queries against the page staged in Kt -> S[(g, query)][key], -inf where not visible
DEVINL void page_scores(const float* qs, const float* Kt, float* S, int c, int rep, int BQ, int D, float scale, int nq,
                        int pos0, int jb) {
  for (int e = threadIdx.x; e < rep * BQ * PAGE; e += 256) {
    const int kj = e % PAGE, r = e / PAGE, qi = r % BQ, g = c * rep + r / BQ;
    const float* qv = qs + ((size_t)g * BQ + qi) * D;
    const float* kv = Kt + kj * (D + 1);
    float s = 0.f;
    for (int d = 0; d < D; ++d) s += qv[d] * kv[d];
    const bool ok = qi < nq && jb + kj <= pos0 + qi;
    S[((size_t)g * BQ + qi) * PAGE + kj] = ok ? s * scale : -INFINITY;
  }
}

template <typename T>
DEVINL void stage_keys(const T* kp, float* Kt, int D) {
  for (int i = threadIdx.x; i < PAGE * D; i += 256) Kt[(i / D) * (D + 1) + i % D] = ldf<T>(kp, i);
}

template <typename T, bool OUT>
__global__ void __launch_bounds__(256) mixed_attn_kernel(
    const T* __restrict__ q, const T* __restrict__ kcache, const T* __restrict__ vcache,
    const int* __restrict__ block_tables, int max_pages, const int* __restrict__ cu_q, const int* __restrict__ ctx_len,
    const T* __restrict__ mix, float* __restrict__ part_ml, T* __restrict__ out, int64_t out_stride,
    float* __restrict__ part_acc, MixShape sh, float scale, float out_scale, int nsplit) {
  extern __shared__ float lds[];
  const int H = sh.H, G = sh.G, D = sh.D, V = sh.V, BQ = sh.BQ;
  const int b = blockIdx.y, split = blockIdx.z, tid = threadIdx.x;
  const int q0 = cu_q[b], qlen = cu_q[b + 1] - q0;
  const int t0 = blockIdx.x * BQ;
  if (t0 >= qlen) return;
  const int nq = min(BQ, qlen - t0);
  const int pos0 = ctx_len[b] - qlen + t0;  // position of the tile's first query
  const int R = H * BQ, rep = H / G;
  float* qs = lds;                           // [H][BQ][D]
  float* Kt = qs + (size_t)R * D;            // [32][D + 1]
  float* S1 = Kt + PAGE * (D + 1);           // [H][BQ][32] scores, then each head's own weights
  float* mrow = S1 + (size_t)R * PAGE;       // [R] running maximum, or the final one
  float* lrow = mrow + R;                    // [R] running sum, or 1 / the final one
  float* S2 = lrow + R;                      // [H][BQ][32] mixed weights
  float* acc = S2 + (size_t)R * PAGE;        // [H][BQ][V]
  float* Vt = acc + (size_t)R * V;           // [V][33]
  float* mixs = Vt + (size_t)V * (PAGE + 1); // [H][H]

  for (int i = tid; i < R * D; i += 256) {
    const int d = i % D, r = i / D, qi = r % BQ, g = r / BQ;
    qs[i] = qi < nq ? ldf<T>(q, ((size_t)(q0 + t0 + qi) * H + g) * D + d) : 0.f;
  }
  for (int i = tid; i < R; i += 256) {
    float m = -1e30f, l = 0.f;
    const int qi = i % BQ, g = i / BQ;
    if (OUT && qi < nq) {
      const float* ml = part_ml + ((size_t)(q0 + t0 + qi) * nsplit * H + g) * 2;
      for (int s = 0; s < nsplit; ++s) m = fmaxf(m, ml[(size_t)s * H * 2]);
      for (int s = 0; s < nsplit; ++s) l += expf(ml[(size_t)s * H * 2] - m) * ml[(size_t)s * H * 2 + 1];
      l = l > 0.f ? 1.f / l : 0.f;
    }
    mrow[i] = m;
    lrow[i] = l;
  }
  if (OUT) {
    for (int i = tid; i < R * V; i += 256) acc[i] = 0.f;
    for (int i = tid; i < H * H; i += 256) mixs[i] = ldf<T>(mix, i);
  }
  const int j_hi = pos0 + nq;
  const int n_pages = (j_hi + PAGE - 1) / PAGE;
  const int per = (n_pages + nsplit - 1) / nsplit;
  const int p_lo = split * per, p_hi = min(n_pages, p_lo + per);

  for (int pg = p_lo; pg < p_hi; ++pg) {
    const size_t page = (size_t)block_tables[(size_t)b * max_pages + pg];
    const int jb = pg * PAGE;
    for (int c = 0; c < G; ++c) {
      __syncthreads();  // Kt free (first time: the tile set-up is visible)
      stage_keys<T>(kcache + ((page * G + c) * PAGE) * D, Kt, D);
      __syncthreads();
      page_scores(qs, Kt, S1, c, rep, BQ, D, scale, nq, pos0, jb);
    }
    __syncthreads();
    // every (head, query) row: 32 lanes a row
    for (int r = tid >> 5; r < R; r += 8) {
      const float s = S1[(size_t)r * PAGE + (tid & 31)];
      if (OUT) {
        S1[(size_t)r * PAGE + (tid & 31)] = expf(s - mrow[r]) * lrow[r];
      } else {
        float mx = s;
#pragma unroll
        for (int o = 16; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
        const float m_old = mrow[r], m_new = fmaxf(m_old, mx);
        float sum = expf(s - m_new);
#pragma unroll
        for (int o = 16; o > 0; o >>= 1) sum += __shfl_xor(sum, o, 64);
        if ((tid & 31) == 0) {
          lrow[r] = lrow[r] * expf(m_old - m_new) + sum;
          mrow[r] = m_new;
        }
      }
    }
    if (!OUT) continue;
    __syncthreads();
    for (int e = tid; e < R * PAGE; e += 256) {
      const int kj = e % PAGE, r = e / PAGE, qi = r % BQ, h = r / BQ;
      float s = 0.f;
      for (int g = 0; g < H; ++g) s += mixs[h * H + g] * S1[((size_t)g * BQ + qi) * PAGE + kj];
      S2[e] = s;
    }
    for (int c = 0; c < G; ++c) {
      __syncthreads();  // Vt free; mixed weights visible
      const T* vp = vcache + ((page * G + c) * V) * PAGE;
      for (int i = tid; i < V * PAGE; i += 256)
        Vt[(i / PAGE) * (PAGE + 1) + i % PAGE] = jb + i % PAGE < j_hi ? ldf<T>(vp, i) : 0.f;
      __syncthreads();
      for (int o = tid; o < rep * BQ * V; o += 256) {
        const int v = o % V, r = c * rep * BQ + o / V;  // heads of a group are consecutive
        const float* pw = S2 + (size_t)r * PAGE;
        float a = acc[(size_t)r * V + v];
#pragma unroll 8
        for (int kj = 0; kj < PAGE; ++kj) a += pw[kj] * Vt[v * (PAGE + 1) + kj];
        acc[(size_t)r * V + v] = a;
      }
    }
  }
  __syncthreads();
  if (!OUT) {
    for (int r = tid; r < R; r += 256) {
      const int qi = r % BQ, g = r / BQ;
      if (qi >= nq) continue;
      float* ml = part_ml + (((size_t)(q0 + t0 + qi) * nsplit + split) * H + g) * 2;
      ml[0] = mrow[r];
      ml[1] = lrow[r];
    }
    return;
  }
  for (int o = tid; o < R * V; o += 256) {
    const int v = o % V, r = o / V, qi = r % BQ, h = r / BQ;
    if (qi >= nq) continue;
    const size_t tok = (size_t)(q0 + t0 + qi);
    if (nsplit == 1) stf<T>(out, tok * out_stride + (size_t)h * V + v, acc[o] * out_scale);
    else part_acc[((tok * nsplit + split) * H + h) * V + v] = acc[o];
  }
}

// one workgroup per (token, 256 output columns): the splits' partial sums are added up
template <typename T>
__global__ void __launch_bounds__(256) mixed_attn_sum_kernel(const float* __restrict__ part_acc, T* __restrict__ out,
                                                             int64_t out_stride, int HV, int nsplit, float out_scale) {
  const size_t tok = blockIdx.x;
  const int i = blockIdx.y * 256 + threadIdx.x;
  if (i >= HV) return;
  float a = 0.f;
  for (int s = 0; s < nsplit; ++s) a += part_acc[(tok * nsplit + s) * HV + i];
  stf<T>(out, tok * out_stride + i, a * out_scale);
}

// ------------------------------------------------------------------------------------------------------------------
// Matrix-core versions (bf16, D and V 64 or 128). Operands come straight from the pages in the order the 16x16x32 MFMA
// wants them: S^T[key, query] = K Q^T with a page's 32 keys as two 16-row tiles whose rows are keys {8c + r} and {8c + 4 + r}
// (c = row / 4, r = row % 4), so that a lane ends up with keys 8 quad .. 8 quad + 7 of its query - the order in which
// O^T[v, query] += V^T P^T reads them. Weights that meet bf16 operands do so as the pair (bf16(w), bf16(w - bf16(w))): 16
// bits of mantissa.

typedef short s16x4 __attribute__((ext_vector_type(4)));

DEVINL f32x4 mfma16(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
DEVINL int key_row(int r16) { return 8 * (r16 >> 2) + (r16 & 3); }

// Prompt portions, first pass: log2 of every (query, head)'s sum of exponentials (log2-scaled scores) -> lse [T, H]. A wave
// serves HPW heads and 16 queries, keeps the running (maximum, sum) per lane over the keys that fall to the lane, and merges
// the four lanes of a query at the end. The next page's keys are fetched under the current one's work. SHARED: the wave's
// heads read one key head.
template <int DK, bool SHARED, int HPW>
__global__ void __launch_bounds__(512, 2) mixed_lse_kernel(
    const bf16_t* __restrict__ q, const bf16_t* __restrict__ kcache, const int* __restrict__ block_tables, int max_pages,
    const int* __restrict__ cu_q, const int* __restrict__ ctx_len, float* __restrict__ lse, int H, int G, float scale_log2) {
  constexpr int D = 32 * DK;
  const int b = blockIdx.x, tile = gridDim.y - 1 - blockIdx.y;  // the tiles with most keys first
  const int q0 = cu_q[b], qlen = cu_q[b + 1] - q0, t0 = tile * 16;
  if (t0 >= qlen) return;
  const int lane = threadIdx.x & 63, r16 = lane & 15, quad = lane >> 4, rep = H / G;
  const int h0 = HPW * (blockIdx.z * (blockDim.x >> 6) + (threadIdx.x >> 6));  // first head of the wave
  const int pos0 = ctx_len[b] - qlen + t0, nq = min(16, qlen - t0), tok = q0 + t0 + min(r16, nq - 1);
  bf16x8 qf[HPW][DK];
  float m[HPW], l[HPW];
#pragma unroll
  for (int hh = 0; hh < HPW; ++hh) {
    m[hh] = -1e30f;
    l[hh] = 0.f;
#pragma unroll
    for (int ks = 0; ks < DK; ++ks) qf[hh][ks] = ld8(q + ((size_t)tok * H + h0 + hh) * D + 32 * ks + 8 * quad);
  }
  const int n_pages = (pos0 + nq + PAGE - 1) / PAGE;
  const int* bt = block_tables + (size_t)b * max_pages;
  const int row_off = key_row(r16) * D + 8 * quad;
  auto load_keys = [&](bf16x8 (&k)[2][DK], int page, int c) {
    const bf16_t* kp = kcache + ((size_t)page * G + c) * PAGE * D + row_off;
#pragma unroll
    for (int ks = 0; ks < DK; ++ks) {
      k[0][ks] = ld8(kp + 32 * ks);
      k[1][ks] = ld8(kp + 4 * D + 32 * ks);
    }
  };
  auto page_step = [&](bf16x8 (&k)[2][DK], int pg, int page) {
    const int jb = pg * PAGE;
    const bool edge = jb + PAGE - 1 > pos0;  // some query of the tile does not see the whole page
#pragma unroll
    for (int hh = 0; hh < HPW; ++hh) {
      if (!SHARED && hh > 0) load_keys(k, page, (h0 + hh) / rep);
      f32x4 sa = {0.f, 0.f, 0.f, 0.f}, sb = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < DK; ++ks) {
        sa = mfma16(k[0][ks], qf[hh][ks], sa);
        sb = mfma16(k[1][ks], qf[hh][ks], sb);
      }
      float s[8];
#pragma unroll
      for (int r = 0; r < 8; ++r) s[r] = (r < 4 ? sa[r & 3] : sb[r & 3]) * scale_log2;
      if (edge) {
        const int last = pos0 + r16 - jb - 8 * quad;  // s[r] is visible for r <= last
#pragma unroll
        for (int r = 0; r < 8; ++r) s[r] = r <= last ? s[r] : -INFINITY;
      }
      const float mx = fmaxf(fmaxf(fmaxf(s[0], s[1]), fmaxf(s[2], s[3])), fmaxf(fmaxf(s[4], s[5]), fmaxf(s[6], s[7])));
      if (__any(mx > m[hh])) {
        const float mn = fmaxf(m[hh], mx);
        l[hh] *= fast_exp2(m[hh] - mn);
        m[hh] = mn;
      }
      float sum = 0.f;
#pragma unroll
      for (int r = 0; r < 8; ++r) sum += fast_exp2(s[r] - m[hh]);
      l[hh] += sum;
    }
  };
  bf16x8 k0[2][DK], k1[2][DK];
  // page ids are fetched ahead of the keys they lead to
  int id0 = bt[0], id1 = bt[min(1, n_pages - 1)], id2 = bt[min(2, n_pages - 1)];
  load_keys(k0, id0, h0 / rep);
  for (int pg = 0; pg < n_pages; pg += 2) {
    const int id3 = bt[min(pg + 3, n_pages - 1)], id4 = bt[min(pg + 4, n_pages - 1)];
    if (pg + 1 < n_pages) load_keys(k1, id1, h0 / rep);
    page_step(k0, pg, id0);
    if (pg + 1 >= n_pages) break;
    if (pg + 2 < n_pages) load_keys(k0, id2, h0 / rep);
    page_step(k1, pg + 1, id1);
    id0 = id2;
    id1 = id3;
    id2 = id4;
  }
#pragma unroll
  for (int hh = 0; hh < HPW; ++hh) {
    const float mm = max_xor32(max_xor16(m[hh]));
    const float ll = sum_xor32(sum_xor16(l[hh] * fast_exp2(m[hh] - mm)));
    if (quad == 0 && r16 < nq) lse[(size_t)tok * H + h0 + hh] = mm + __log2f(ll);
  }
}

// Prompt portions, second pass. One workgroup = 16 queries x all H heads, wave w owning heads HPW w .. HPW w + HPW - 1. Per
// page:
//   weights  p of the owned heads in registers (lane: query r16, keys 8 quad + j), their (hi, lo) halves into LDS next to
//            the other waves': [j][16-byte piece][lane], a piece holding 8 heads' halves of one (query, key)
//   mix      v_mfma_f32_4x4x4 (16 blocks): every lane's own (query, key) against the owned rows of M - no data crosses lanes
//   values   O^T += V^T W^T per owned head, two products (hi, lo)
// The weights' LDS buffer is double: one barrier a page. Keys of the next page are fetched ahead.
template <int DK, int VT, bool SHARED, int NW, int HPW>
__global__ void __launch_bounds__(64 * NW, (NW * HPW == 16 && HPW == 4 ? 1 : 2)) mixed_apply_kernel(
    const bf16_t* __restrict__ q, const bf16_t* __restrict__ kcache, const bf16_t* __restrict__ vcache,
    const int* __restrict__ block_tables, int max_pages, const int* __restrict__ cu_q, const int* __restrict__ ctx_len,
    const bf16_t* __restrict__ mix, const float* __restrict__ lse, bf16_t* __restrict__ out, int64_t out_stride, int G,
    float scale_log2, float out_scale) {
  constexpr int D = 32 * DK, V = 16 * VT, H = HPW * NW, NP = (H + 7) / 8;  // 16-byte pieces of the hi (and lo) halves
  // registers left for the next page's keys (four waves a workgroup, one a SIMD: all of the register file)
  constexpr bool AHEAD = SHARED && (HPW * (8 * VT / 2 + 4 * DK) < 160 || NW == 4);
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int b = blockIdx.x, tile = gridDim.y - 1 - blockIdx.y;
  const int q0 = cu_q[b], qlen = cu_q[b + 1] - q0, t0 = tile * 16;
  if (t0 >= qlen) return;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, r16 = lane & 15, quad = lane >> 4, rep = H / G;
  const int nq = min(16, qlen - t0), pos0 = ctx_len[b] - qlen + t0, tok = q0 + t0 + min(r16, nq - 1);
  bf16x8 qf[HPW][DK];
  float ls[HPW];
  f32x4 acc[HPW][VT];
#pragma unroll
  for (int hh = 0; hh < HPW; ++hh) {
    ls[hh] = r16 < nq ? lse[(size_t)tok * H + HPW * w + hh] : INFINITY;  // rows past the tile weigh nothing
#pragma unroll
    for (int ks = 0; ks < DK; ++ks) qf[hh][ks] = ld8(q + ((size_t)tok * H + HPW * w + hh) * D + 32 * ks + 8 * quad);
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) acc[hh][vt] = (f32x4){0.f, 0.f, 0.f, 0.f};
  }
  s16x4 mf[H / 4];  // the owned rows of M, row lane & 3 in this lane (rows past HPW repeat)
#pragma unroll
  for (int gg = 0; gg < H / 4; ++gg)
    mf[gg] = *reinterpret_cast<const s16x4*>(mix + (size_t)(HPW * w + (lane & (HPW - 1))) * H + 4 * gg);
  const int j_hi = pos0 + nq, n_pages = (j_hi + PAGE - 1) / PAGE;
  const int* bt = block_tables + (size_t)b * max_pages;
  const int row_off = key_row(r16) * D + 8 * quad;
  bf16x8 k[2][DK];
  auto load_keys = [&](int id, int c) {
    const bf16_t* kp = kcache + ((size_t)id * G + c) * PAGE * D + row_off;
#pragma unroll
    for (int ks = 0; ks < DK; ++ks) {
      k[0][ks] = ld8(kp + 32 * ks);
      k[1][ks] = ld8(kp + 4 * D + 32 * ks);
    }
  };
  int id = bt[0], id_next = bt[min(1, n_pages - 1)];  // page ids are fetched ahead of what they lead to
  if (AHEAD) load_keys(id, HPW * w / rep);
  for (int pg = 0; pg < n_pages; ++pg) {
    char* buf = smem + (pg & 1) * (8 * 2 * NP * 64 * 16);
    const int id_after = bt[min(pg + 2, n_pages - 1)];
    const size_t page = (size_t)id * G;
    const int jb = pg * PAGE;
    float p[HPW][8];
#pragma unroll
    for (int hh = 0; hh < HPW; ++hh) {
      if (!AHEAD && (hh == 0 || !SHARED)) load_keys(id, (HPW * w + hh) / rep);
      f32x4 sa = {0.f, 0.f, 0.f, 0.f}, sb = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < DK; ++ks) {
        sa = mfma16(k[0][ks], qf[hh][ks], sa);
        sb = mfma16(k[1][ks], qf[hh][ks], sb);
      }
#pragma unroll
      for (int r = 0; r < 8; ++r) p[hh][r] = fast_exp2((r < 4 ? sa[r & 3] : sb[r & 3]) * scale_log2 - ls[hh]);
    }
    bf16x8 vf[VT];
    auto load_values = [&](int c) {
      const bf16_t* vp = vcache + (page + c) * V * PAGE;
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) vf[vt] = ld8(vp + (16 * vt + r16) * PAGE + 8 * quad);
      if (jb + PAGE > j_hi) {  // page slots past the last key may hold anything
        const int live = j_hi - jb - 8 * quad;
#pragma unroll
        for (int vt = 0; vt < VT; ++vt)
#pragma unroll
          for (int e = 0; e < 8; ++e) vf[vt][e] = e < live ? vf[vt][e] : (bf16_t)0.f;
      }
    };
    if (SHARED) load_values(HPW * w / rep);
    if (AHEAD && pg + 1 < n_pages) load_keys(id_next, HPW * w / rep);
    if (jb + PAGE - 1 > pos0) {
      const int last = pos0 + r16 - jb - 8 * quad;
#pragma unroll
      for (int hh = 0; hh < HPW; ++hh)
#pragma unroll
        for (int r = 0; r < 8; ++r) p[hh][r] = r <= last ? p[hh][r] : 0.f;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      typedef bf16_t half_t __attribute__((ext_vector_type(HPW)));
      half_t hi, lo;
#pragma unroll
      for (int hh = 0; hh < HPW; ++hh) {
        hi[hh] = f2bf(p[hh][j]);
        lo[hh] = f2bf(p[hh][j] - bf2f(hi[hh]));
      }
      char* at = buf + (((j * 2 * NP + (HPW * w >> 3)) * 64 + lane) * 16 + 2 * (HPW * w & 7));
      *reinterpret_cast<half_t*>(at) = hi;
      *reinterpret_cast<half_t*>(at + NP * 64 * 16) = lo;
    }
    __syncthreads();  // everybody's weights of this page are in LDS
    bf16x8 wh[HPW], wl[HPW];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      f32x4 c0 = {0.f, 0.f, 0.f, 0.f}, c1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int pc = 0; pc < NP; ++pc) {
        const char* at = buf + ((j * 2 * NP + pc) * 64 + lane) * 16;
        const bf16x8 h8 = *reinterpret_cast<const bf16x8*>(at), l8 = *reinterpret_cast<const bf16x8*>(at + NP * 64 * 16);
        const bf16x4 h0 = {h8[0], h8[1], h8[2], h8[3]}, l0 = {l8[0], l8[1], l8[2], l8[3]};
        c0 = __builtin_amdgcn_mfma_f32_4x4x4bf16_1k(mf[2 * pc], __builtin_bit_cast(s16x4, h0), c0, 0, 0, 0);
        c1 = __builtin_amdgcn_mfma_f32_4x4x4bf16_1k(mf[2 * pc], __builtin_bit_cast(s16x4, l0), c1, 0, 0, 0);
        if (2 * pc + 1 < H / 4) {
          const bf16x4 h1 = {h8[4], h8[5], h8[6], h8[7]}, l1 = {l8[4], l8[5], l8[6], l8[7]};
          c0 = __builtin_amdgcn_mfma_f32_4x4x4bf16_1k(mf[2 * pc + 1], __builtin_bit_cast(s16x4, h1), c0, 0, 0, 0);
          c1 = __builtin_amdgcn_mfma_f32_4x4x4bf16_1k(mf[2 * pc + 1], __builtin_bit_cast(s16x4, l1), c1, 0, 0, 0);
        }
      }
      c0 += c1;
#pragma unroll
      for (int hh = 0; hh < HPW; ++hh) {
        wh[hh][j] = f2bf(c0[hh]);
        wl[hh][j] = f2bf(c0[hh] - bf2f(wh[hh][j]));
      }
    }
#pragma unroll
    for (int hh = 0; hh < HPW; ++hh) {
      if (!SHARED) load_values((HPW * w + hh) / rep);
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) acc[hh][vt] = mfma16(vf[vt], wh[hh], acc[hh][vt]);
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) acc[hh][vt] = mfma16(vf[vt], wl[hh], acc[hh][vt]);
    }
    id = id_next;
    id_next = id_after;
  }
  if (r16 < nq) {
#pragma unroll
    for (int hh = 0; hh < HPW; ++hh)
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) {
        bf16x4 o;
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] = f2bf(acc[hh][vt][i] * out_scale);
        *reinterpret_cast<bf16x4*>(out + (size_t)tok * out_stride + (size_t)(HPW * w + hh) * V + 16 * vt + 4 * quad) = o;
      }
  }
}

// Decoding (one query per row), first pass: grid (row, key/value head, split), four waves, a page a wave and step. Leaves
// the log2-scaled scores in sc [row, H, n_keys] (-inf past the context) and (maximum, sum) per (row, split, head).
template <int DK>
__global__ void __launch_bounds__(256) mixed_decode_scores_kernel(
    const bf16_t* __restrict__ q, const bf16_t* __restrict__ kcache, const int* __restrict__ block_tables, int max_pages,
    const int* __restrict__ ctx_len, float* __restrict__ sc, int64_t n_keys, float* __restrict__ part_ml, int H, int G,
    float scale_log2) {
  constexpr int D = 32 * DK;
  __shared__ float sm[4][16], sl[4][16];
  const int b = blockIdx.x, c = blockIdx.y, split = blockIdx.z, nsplit = gridDim.z;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, r16 = lane & 15, quad = lane >> 4, rep = H / G;
  const int ctx = ctx_len[b], n_pages = (ctx + PAGE - 1) / PAGE, per = (n_pages + nsplit - 1) / nsplit;
  const int p_lo = split * per, p_hi = min(n_pages, p_lo + per);
  const int head = c * rep + min(r16, rep - 1);
  bf16x8 qf[DK];
#pragma unroll
  for (int ks = 0; ks < DK; ++ks) qf[ks] = ld8(q + ((size_t)b * H + head) * D + 32 * ks + 8 * quad);
  float m = -1e30f, l = 0.f;
  for (int pg = p_lo + w; pg < p_hi; pg += 4) {
    const bf16_t* kp = kcache + ((size_t)block_tables[(size_t)b * max_pages + pg] * G + c) * PAGE * D;
    bf16x8 ka[DK], kb[DK];
#pragma unroll
    for (int ks = 0; ks < DK; ++ks) {
      ka[ks] = ld8(kp + key_row(r16) * D + 32 * ks + 8 * quad);
      kb[ks] = ld8(kp + (key_row(r16) + 4) * D + 32 * ks + 8 * quad);
    }
    f32x4 sa = {0.f, 0.f, 0.f, 0.f}, sb = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < DK; ++ks) {
      sa = mfma16(ka[ks], qf[ks], sa);
      sb = mfma16(kb[ks], qf[ks], sb);
    }
    const int key0 = pg * PAGE + 8 * quad;
    float mx = m;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      sa[r] = key0 + r < ctx ? sa[r] * scale_log2 : -INFINITY;
      sb[r] = key0 + 4 + r < ctx ? sb[r] * scale_log2 : -INFINITY;
      mx = fmaxf(mx, fmaxf(sa[r], sb[r]));
    }
    l *= fast_exp2(m - mx);
    m = mx;
#pragma unroll
    for (int r = 0; r < 4; ++r) l += fast_exp2(sa[r] - m) + fast_exp2(sb[r] - m);
    if (r16 < rep) {
      float* dst = sc + ((size_t)b * H + head) * n_keys + key0;
      *reinterpret_cast<f32x4*>(dst) = sa;
      *reinterpret_cast<f32x4*>(dst + 4) = sb;
    }
  }
  const float mm = max_xor32(max_xor16(m));
  const float ll = sum_xor32(sum_xor16(l * fast_exp2(m - mm)));
  if (quad == 0) {
    sm[w][r16] = mm;
    sl[w][r16] = ll;
  }
  __syncthreads();
  if (threadIdx.x < rep) {
    const int i = threadIdx.x;
    const float M = fmaxf(fmaxf(sm[0][i], sm[1][i]), fmaxf(sm[2][i], sm[3][i]));
    float L = 0.f;
#pragma unroll
    for (int k = 0; k < 4; ++k) L += sl[k][i] * fast_exp2(sm[k][i] - M);
    float* ml = part_ml + (((size_t)b * nsplit + split) * H + c * rep + i) * 2;
    ml[0] = M;
    ml[1] = L;
  }
}

// Decoding, second pass: the same grid; c is the value head whose rep heads the workgroup serves. A page's weights of all
// heads are mixed on the fp32 matrix cores (16x16x4: rows = keys in the order of `key_row`, k = heads, columns = this
// group's heads), so a lane ends up with its head's weights of keys 8 quad .. 8 quad + 7. HK: number of k-steps, H <= 4 HK.
template <int VT, int HK>
__global__ void __launch_bounds__(256) mixed_decode_values_kernel(
    const bf16_t* __restrict__ vcache, const int* __restrict__ block_tables, int max_pages, const int* __restrict__ ctx_len,
    const bf16_t* __restrict__ mix, const float* __restrict__ sc, int64_t n_keys, const float* __restrict__ part_ml,
    bf16_t* __restrict__ out, int64_t out_stride, float* __restrict__ part_acc, int H, int G, float out_scale) {
  constexpr int V = 16 * VT, VS = V + 4;
  __shared__ __attribute__((aligned(16))) float so[4][16][VS];
  __shared__ float slse[4 * HK];
  const int b = blockIdx.x, c = blockIdx.y, split = blockIdx.z, nsplit = gridDim.z, tid = threadIdx.x;
  const int lane = tid & 63, w = tid >> 6, r16 = lane & 15, quad = lane >> 4, rep = H / G;
  const int ctx = ctx_len[b], n_pages = (ctx + PAGE - 1) / PAGE, per = (n_pages + nsplit - 1) / nsplit;
  const int p_lo = split * per, p_hi = min(n_pages, p_lo + per);
  for (int g = tid; g < 4 * HK; g += 256) {
    float m = -1e30f, l = 0.f;
    if (g < H) {
      const float* ml = part_ml + ((size_t)b * nsplit * H + g) * 2;
      for (int s = 0; s < nsplit; ++s) m = fmaxf(m, ml[(size_t)s * H * 2]);
      for (int s = 0; s < nsplit; ++s) l += fast_exp2(ml[(size_t)s * H * 2] - m) * ml[(size_t)s * H * 2 + 1];
    }
    slse[g] = l > 0.f ? m + __log2f(l) : INFINITY;
  }
  __syncthreads();
  float mt[HK], ls[HK];  // M[this lane's head, head 4 kk + quad], and that head's log2 sum
#pragma unroll
  for (int kk = 0; kk < HK; ++kk) {
    const int g = 4 * kk + quad;
    mt[kk] = (r16 < rep && g < H) ? bf2f(mix[(size_t)(c * rep + r16) * H + g]) : 0.f;
    ls[kk] = slse[g];
  }
  f32x4 acc[VT];
#pragma unroll
  for (int vt = 0; vt < VT; ++vt) acc[vt] = (f32x4){0.f, 0.f, 0.f, 0.f};
  for (int pg = p_lo + w; pg < p_hi; pg += 4) {
    const bf16_t* vp = vcache + ((size_t)block_tables[(size_t)b * max_pages + pg] * G + c) * V * PAGE;
    bf16x8 vf[VT];
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) vf[vt] = ld8(vp + (16 * vt + r16) * PAGE + 8 * quad);
    const int jb = pg * PAGE;
    float xa[HK], xb[HK];
#pragma unroll
    for (int kk = 0; kk < HK; ++kk) {
      const float* src = sc + ((size_t)b * H + min(4 * kk + quad, H - 1)) * n_keys + jb + key_row(r16);
      xa[kk] = src[0];
      xb[kk] = src[4];
    }
    if (jb + PAGE > ctx) {
      const int live = ctx - jb - 8 * quad;
#pragma unroll
      for (int vt = 0; vt < VT; ++vt)
#pragma unroll
        for (int e = 0; e < 8; ++e) vf[vt][e] = e < live ? vf[vt][e] : (bf16_t)0.f;
    }
    f32x4 wa = {0.f, 0.f, 0.f, 0.f}, wb = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < HK; ++kk) {
      wa = __builtin_amdgcn_mfma_f32_16x16x4f32(fast_exp2(xa[kk] - ls[kk]), mt[kk], wa, 0, 0, 0);
      wb = __builtin_amdgcn_mfma_f32_16x16x4f32(fast_exp2(xb[kk] - ls[kk]), mt[kk], wb, 0, 0, 0);
    }
    bf16x8 wh, wl;
#pragma unroll
    for (int r = 0; r < 8; ++r) {
      const float x = r < 4 ? wa[r & 3] : wb[r & 3];
      wh[r] = f2bf(x);
      wl[r] = f2bf(x - bf2f(wh[r]));
    }
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) {
      acc[vt] = mfma16(vf[vt], wh, acc[vt]);
      acc[vt] = mfma16(vf[vt], wl, acc[vt]);
    }
  }
  if (r16 < rep) {
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) *reinterpret_cast<f32x4*>(&so[w][r16][16 * vt + 4 * quad]) = acc[vt];
  }
  __syncthreads();
  for (int i = tid; i < rep * V; i += 256) {
    const int hl = i / V, v = i % V, h = c * rep + hl;
    const float a = so[0][hl][v] + so[1][hl][v] + so[2][hl][v] + so[3][hl][v];
    if (nsplit == 1) out[(size_t)b * out_stride + (size_t)h * V + v] = f2bf(a * out_scale);
    else part_acc[(((size_t)b * nsplit + split) * H + h) * V + v] = a;
  }
}

bool matrix_sizes(int D, int V) { return (D == 64 || D == 128) && (V == 64 || V == 128); }

}  // namespace

// Largest query tile (at most `want`) of the any-size kernel whose LDS footprint fits; 0 if even one query does not.
extern "C" int areal_mixed_attn_tile(int H, int G, int D, int V, int want) {
  for (int bq = want; bq >= 1; bq >>= 1) {
    MixShape sh{H, G, D, V, bq};
    if (sh.floats() * sizeof(float) <= 156 * 1024) return bq;
  }
  return 0;
}

// B rows; row b's queries are tokens cu_q[b] .. cu_q[b+1] of q [T, H, D]; max_q = longest row. out rows of H V numbers,
// out_stride apart. part_ml [T, nsplit, H, 2] fp32 always; nsplit > 1 (single-query rows) also part_acc [T, nsplit, H, V].
extern "C" int areal_mixed_attn(const void* q, const void* kcache, const void* vcache, const int* block_tables,
                                int max_pages, const int* cu_q, const int* ctx_len, const void* mix, float* part_ml,
                                void* out, int64_t out_stride, float* part_acc, int B, int max_q, int T, int H, int G,
                                int D, int V, int bq, float scale, float out_scale, int nsplit, int dt, hipStream_t st) {
  if (B == 0 || T == 0) return 0;
  if (G <= 0 || H % G != 0 || bq <= 0 || nsplit < 1 || !part_ml || !mix) return -1;
  MixShape sh{H, G, D, V, bq};
  const size_t lds = sh.floats() * sizeof(float);
  if (lds > 160 * 1024) return -2;
  if (nsplit > 1 && (!part_acc || max_q != 1)) return -3;
  const dim3 grid((max_q + bq - 1) / bq, B, nsplit);
#define LAUNCH(TT)                                                                                                    \
  do {                                                                                                                \
    static bool raised = false; /* once: no attribute call inside a stream capture later */                           \
    if (!raised) {                                                                                                    \
      HIP_RET(hipFuncSetAttribute((const void*)mixed_attn_kernel<TT, false>,                                          \
                                  hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));                           \
      HIP_RET(hipFuncSetAttribute((const void*)mixed_attn_kernel<TT, true>,                                           \
                                  hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));                           \
      raised = true;                                                                                                  \
    }                                                                                                                 \
    hipLaunchKernelGGL((mixed_attn_kernel<TT, false>), grid, dim3(256), lds, st, (const TT*)q, (const TT*)kcache,     \
                       (const TT*)vcache, block_tables, max_pages, cu_q, ctx_len, (const TT*)mix, part_ml, (TT*)out,  \
                       out_stride, part_acc, sh, scale, out_scale, nsplit);                                           \
    hipLaunchKernelGGL((mixed_attn_kernel<TT, true>), grid, dim3(256), lds, st, (const TT*)q, (const TT*)kcache,      \
                       (const TT*)vcache, block_tables, max_pages, cu_q, ctx_len, (const TT*)mix, part_ml, (TT*)out,  \
                       out_stride, part_acc, sh, scale, out_scale, nsplit);                                           \
    if (nsplit > 1)                                                                                                   \
      hipLaunchKernelGGL(mixed_attn_sum_kernel<TT>, dim3(T, (H * V + 255) / 256), dim3(256), 0, st, part_acc,         \
                         (TT*)out, out_stride, H * V, nsplit, out_scale);                                             \
  } while (0)
  if (dt == 0) LAUNCH(bf16_t);
  else LAUNCH(float);
#undef LAUNCH
  return (int)hipGetLastError();
}

// Whether the matrix-core kernels serve these sizes: bit 0 prompt portions, bit 1 decoding (bf16 storage only).
extern "C" int areal_mixed_attn_matrix_cores(int H, int G, int D, int V) {
  if (G <= 0 || H <= 0 || H % G != 0 || !matrix_sizes(D, V)) return 0;
  const bool prompt = H == 4 || H == 8 || H == 16 || H == 32;
  const bool decode = H / G <= 16 && H <= 64;
  return (prompt ? 1 : 0) | (decode ? 2 : 0);
}

// Prompt portions on the matrix cores: lse [T, H] fp32 is scratch; out rows 8-byte aligned.
extern "C" int areal_mixed_attn_prompt(const void* q, const void* kcache, const void* vcache, const int* block_tables,
                                       int max_pages, const int* cu_q, const int* ctx_len, const void* mix, float* lse,
                                       void* out, int64_t out_stride, int B, int max_q, int T, int H, int G, int D, int V,
                                       float scale, float out_scale, hipStream_t st) {
  if (B == 0 || T == 0) return 0;
  if (!(areal_mixed_attn_matrix_cores(H, G, D, V) & 1) || !lse) return -1;
  if (out_stride % 4 != 0 || (uintptr_t)out % 8 != 0 || (uintptr_t)mix % 8 != 0) return -2;
  if ((max_q + 15) / 16 > 65535) return -3;
  const float s2 = scale * LOG2E;
  // heads per wave of the second pass; at 16 heads four of one key head: a page's keys and values are loaded once
  const int hpw = H == 32 || (H == 16 && (H / G) % 4 == 0) ? 4 : 2, nw = H / hpw;
  const bool shared = (H / G) % hpw == 0;
  const size_t lds = (size_t)2 * 8 * 2 * ((H + 7) / 8) * 64 * 16;
  // the first pass: four heads a wave where they read one key head (a page's keys are loaded once), else two
#define STATS_W(DKV, SH, HW)                                                                                         \
  hipLaunchKernelGGL((mixed_lse_kernel<DKV, SH, HW>), dim3(B, (max_q + 15) / 16, (H / HW + 7) / 8),                    \
                     dim3(64 * (H / HW < 8 ? H / HW : 8)), 0, st, (const bf16_t*)q, (const bf16_t*)kcache,            \
                     block_tables, max_pages, cu_q, ctx_len, lse, H, G, s2)
#define STATS(DKV)                                       \
  do {                                                   \
    if ((H / G) % 4 == 0) STATS_W(DKV, true, 4);         \
    else if ((H / G) % 2 == 0) STATS_W(DKV, true, 2);    \
    else STATS_W(DKV, false, 2);                         \
  } while (0)
  if (D == 128) STATS(4);
  else STATS(2);
#undef STATS_W
#undef STATS
#define APPLY(DKV, VTV, SH, NWV, HPWV)                                                                              \
  do {                                                                                                              \
    static bool raised = false;                                                                                     \
    if (!raised && lds > 64 * 1024) {                                                                               \
      HIP_RET(hipFuncSetAttribute((const void*)mixed_apply_kernel<DKV, VTV, SH, NWV, HPWV>,                         \
                                  hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));                         \
      raised = true;                                                                                                \
    }                                                                                                               \
    hipLaunchKernelGGL((mixed_apply_kernel<DKV, VTV, SH, NWV, HPWV>), dim3(B, (max_q + 15) / 16), dim3(64 * NWV), lds, \
                       st, (const bf16_t*)q, (const bf16_t*)kcache, (const bf16_t*)vcache, block_tables, max_pages, \
                       cu_q, ctx_len, (const bf16_t*)mix, lse, (bf16_t*)out, out_stride, G, s2, out_scale);         \
  } while (0)
#define APPLY_NW(DKV, VTV, SH)                     \
  do {                                             \
    if (nw == 2) APPLY(DKV, VTV, SH, 2, 2);        \
    else if (nw == 4 && hpw == 2) APPLY(DKV, VTV, SH, 4, 2); \
    else if (nw == 4) APPLY(DKV, VTV, SH, 4, 4);   \
    else if (H == 16) APPLY(DKV, VTV, SH, 8, 2);   \
    else APPLY(DKV, VTV, SH, 8, 4);                \
  } while (0)
#define APPLY_SH(DKV, VTV)                 \
  do {                                     \
    if (shared) APPLY_NW(DKV, VTV, true);  \
    else APPLY_NW(DKV, VTV, false);        \
  } while (0)
  if (D == 128 && V == 128) APPLY_SH(4, 8);
  else if (D == 128) APPLY_SH(4, 4);
  else if (V == 128) APPLY_SH(2, 8);
  else APPLY_SH(2, 4);
#undef APPLY_SH
#undef APPLY_NW
#undef APPLY
  return (int)hipGetLastError();
}

// Decoding on the matrix cores: B rows of one query. sc [B, H, 32 max_pages] fp32, part_ml [B, nsplit, H, 2] and (nsplit > 1)
// part_acc [B, nsplit, H, V] fp32 are scratch.
extern "C" int areal_mixed_attn_decode(const void* q, const void* kcache, const void* vcache, const int* block_tables,
                                       int max_pages, const int* ctx_len, const void* mix, float* sc, float* part_ml,
                                       void* out, int64_t out_stride, float* part_acc, int B, int H, int G, int D, int V,
                                       float scale, float out_scale, int nsplit, hipStream_t st) {
  if (B == 0) return 0;
  if (!(areal_mixed_attn_matrix_cores(H, G, D, V) & 2) || !sc || !part_ml || nsplit < 1) return -1;
  if (nsplit > 1 && !part_acc) return -3;
  const float s2 = scale * LOG2E;
  const int64_t n_keys = (int64_t)PAGE * max_pages;
  const dim3 grid(B, G, nsplit);
#define SCORES(DKV)                                                                                               \
  hipLaunchKernelGGL(mixed_decode_scores_kernel<DKV>, grid, dim3(256), 0, st, (const bf16_t*)q, (const bf16_t*)kcache, \
                     block_tables, max_pages, ctx_len, sc, n_keys, part_ml, H, G, s2)
  if (D == 128) SCORES(4);
  else SCORES(2);
#undef SCORES
#define VALUES(VTV, HKV)                                                                                              \
  hipLaunchKernelGGL((mixed_decode_values_kernel<VTV, HKV>), grid, dim3(256), 0, st, (const bf16_t*)vcache, block_tables, \
                     max_pages, ctx_len, (const bf16_t*)mix, sc, n_keys, part_ml, (bf16_t*)out, out_stride, part_acc,  \
                     H, G, out_scale)
#define VALUES_H(VTV)             \
  do {                            \
    if (H <= 8) VALUES(VTV, 2);   \
    else if (H <= 16) VALUES(VTV, 4); \
    else if (H <= 32) VALUES(VTV, 8); \
    else VALUES(VTV, 16);         \
  } while (0)
  if (V == 128) VALUES_H(8);
  else VALUES_H(4);
#undef VALUES_H
#undef VALUES
  if (nsplit > 1)
    hipLaunchKernelGGL(mixed_attn_sum_kernel<bf16_t>, dim3(B, (H * V + 255) / 256), dim3(256), 0, st, part_acc,
                       (bf16_t*)out, out_stride, H * V, nsplit, out_scale);
  return (int)hipGetLastError();
}
