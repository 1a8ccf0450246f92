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
