// Sublayers between two layer norms on an fp32 residual stream, the per-channel causal convolution on a mixer's
// input, and the token + hashed-bigram embedding. One workgroup per token; a token's row is staged in LDS once
// and every statistic is an fp32 sum over it (mean first, then the mean of the squared deviations).
//
//   layer_norm32      h = (x - mean) / sqrt(var + eps) * w + b                          -> fp32 and / or storage type
//   gated_norm_add    x <- x + s * LN(y * sigmoid(r); w, b)   [+ the next sublayer's norm of the new x]
//   canon_conv        out_t = h_t + sum_j w[:, j] h_(t - taps + 1 + j); history before a row's first token comes
//                     from the row's state slot (zeros before position 0); the slot then takes the row's last inputs
//   conv_silu         out_t = silu(sum_j w[:, j] h_(t - taps + 1 + j) + bias), the same history
//   norm_add_conv     xo = x + LN(y; w, b) and xo + conv(xo) in one launch
//   embed_bigram_norm x = LN(E[tok] + B[(prev * a + tok * b) mod n])   (row n of B at position 0)
//
// T is the storage type (bf16 / fp32) of weights and of the sublayers' outputs; the stream x is fp32.
// Rows of the packed batch: row b owns tokens cu_q[b] .. cu_q[b+1], its first token has position first_pos[b], its
// state lives in slot state_slots[b] (negative: a padding row that touches no state).
#include "common.hpp"

namespace {

template <typename T> DEVINL float ldf(const T* p, size_t i);
template <> DEVINL float ldf<bf16_t>(const bf16_t* p, size_t i) { return bf2f(p[i]); }
template <> DEVINL float ldf<float>(const float* p, size_t i) { return p[i]; }
template <typename T> DEVINL void stf(T* p, size_t i, float v);
template <> DEVINL void stf<bf16_t>(bf16_t* p, size_t i, float v) { p[i] = f2bf(v); }
template <> DEVINL void stf<float>(float* p, size_t i, float v) { p[i] = v; }

// Four consecutive elements at index i (a multiple of 4; the pointers are 16-byte aligned and rows are multiples of 4).
template <typename T> DEVINL f32x4 ld4(const T* p, size_t i);
template <> DEVINL f32x4 ld4<bf16_t>(const bf16_t* p, size_t i) {
  const bf16x4 v = *reinterpret_cast<const bf16x4*>(p + i);
  return (f32x4){bf2f(v[0]), bf2f(v[1]), bf2f(v[2]), bf2f(v[3])};
}
template <> DEVINL f32x4 ld4<float>(const float* p, size_t i) { return *reinterpret_cast<const f32x4*>(p + i); }
template <typename T> DEVINL void st4(T* p, size_t i, f32x4 v);
template <> DEVINL void st4<bf16_t>(bf16_t* p, size_t i, f32x4 v) {
  *reinterpret_cast<bf16x4*>(p + i) = (bf16x4){f2bf(v[0]), f2bf(v[1]), f2bf(v[2]), f2bf(v[3])};
}
template <> DEVINL void st4<float>(float* p, size_t i, f32x4 v) { *reinterpret_cast<f32x4*>(p + i) = v; }

// Sum over the threads of a workgroup (a multiple of 64, at most 1024); every thread gets the result. `red` holds 16
// floats. Every thread adds the waves' sums in the same order, so all of them see the same bits.
DEVINL float block_sum(float v, float* red) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
  for (int w = 0; w < (int)(blockDim.x >> 6); ++w) s += red[w];
  return s;
}

// (mean, 1 / sqrt(var + eps)) of the W floats in `row` (LDS); every thread gets both.
DEVINL void row_stats(const float* row, int W, float eps, float* red, float& mean, float& rstd) {
  float s = 0.f;
  for (int i = threadIdx.x; i < W; i += blockDim.x) s += row[i];
  mean = block_sum(s, red) / (float)W;
  float v = 0.f;
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    const float d = row[i] - mean;
    v += d * d;
  }
  rstd = 1.f / sqrtf(block_sum(v, red) / (float)W + eps);
}

// Row of the packed batch that owns token t: cu_q is ascending, cu_q[0] = 0, cu_q[B] >= t + 1 for live tokens.
DEVINL int row_of(const int* __restrict__ cu_q, int B, int t) {
  int lo = 0, hi = B - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (cu_q[mid] <= t) lo = mid;
    else hi = mid - 1;
  }
  return lo;
}

template <typename T, bool V4>
__global__ void __launch_bounds__(1024) layer_norm32_kernel(const float* __restrict__ x, const T* __restrict__ w,
                                                            const T* __restrict__ b, float* __restrict__ o32,
                                                            T* __restrict__ oc, int W, float eps) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  float* red = row + W;
  const size_t base = (size_t)blockIdx.x * W;
  if (V4) {
    for (int i = 4 * threadIdx.x; i < W; i += 4 * blockDim.x) *reinterpret_cast<f32x4*>(row + i) = ld4<float>(x, base + i);
  } else {
    for (int i = threadIdx.x; i < W; i += blockDim.x) row[i] = x[base + i];
  }
  __syncthreads();
  float mean, rstd;
  row_stats(row, W, eps, red, mean, rstd);
  if (V4) {
    for (int i = 4 * threadIdx.x; i < W; i += 4 * blockDim.x) {
      const f32x4 h = (*reinterpret_cast<const f32x4*>(row + i) - mean) * rstd * ld4<T>(w, i) + ld4<T>(b, i);
      if (o32) st4<float>(o32, base + i, h);
      if (oc) st4<T>(oc, base + i, h);
    }
  } else {
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
      const float h = (row[i] - mean) * rstd * ldf<T>(w, i) + ldf<T>(b, i);
      if (o32) o32[base + i] = h;
      if (oc) stf<T>(oc, base + i, h);
    }
  }
}

// V4: rows that are multiples of 4 wide move as 16-byte (fp32) / 8-byte (bf16) vectors.
template <typename T, bool V4>
__global__ void __launch_bounds__(1024) gated_norm_add_kernel(
    float* __restrict__ x, const T* __restrict__ y, const T* __restrict__ gate, const T* __restrict__ w,
    const T* __restrict__ b, const T* __restrict__ scale, const T* __restrict__ nw, const T* __restrict__ nb,
    float* __restrict__ h32, T* __restrict__ hc, int W, float eps) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  float* red = row + W;
  const size_t base = (size_t)blockIdx.x * W;
  if (V4) {
    for (int i = 4 * threadIdx.x; i < W; i += 4 * blockDim.x) {
      f32x4 z = ld4<T>(y, base + i);
      if (gate) {
        const f32x4 g = ld4<T>(gate, base + i);
#pragma unroll
        for (int k = 0; k < 4; ++k) z[k] /= 1.f + expf(-g[k]);
      }
      *reinterpret_cast<f32x4*>(row + i) = z;
    }
  } else {
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
      float z = ldf<T>(y, base + i);
      if (gate) z /= 1.f + expf(-ldf<T>(gate, base + i));
      row[i] = z;
    }
  }
  __syncthreads();
  float mean, rstd;
  row_stats(row, W, eps, red, mean, rstd);
  if (V4) {
    for (int i = 4 * threadIdx.x; i < W; i += 4 * blockDim.x) {
      f32x4 r = (*reinterpret_cast<const f32x4*>(row + i) - mean) * rstd * ld4<T>(w, i) + ld4<T>(b, i);
      if (scale) r *= ld4<T>(scale, i);
      const f32x4 nx = ld4<float>(x, base + i) + r;
      st4<float>(x, base + i, nx);
      *reinterpret_cast<f32x4*>(row + i) = nx;  // the elements this thread owns in every pass
    }
  } else {
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
      float r = (row[i] - mean) * rstd * ldf<T>(w, i) + ldf<T>(b, i);
      if (scale) r *= ldf<T>(scale, i);
      const float nx = x[base + i] + r;
      x[base + i] = nx;
      row[i] = nx;  // the element this thread owns in every pass
    }
  }
  if (!nw) return;
  __syncthreads();
  row_stats(row, W, eps, red, mean, rstd);
  if (V4) {
    for (int i = 4 * threadIdx.x; i < W; i += 4 * blockDim.x) {
      const f32x4 h = (*reinterpret_cast<const f32x4*>(row + i) - mean) * rstd * ld4<T>(nw, i) + ld4<T>(nb, i);
      if (h32) st4<float>(h32, base + i, h);
      if (hc) st4<T>(hc, base + i, h);
    }
  } else {
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
      const float h = (row[i] - mean) * rstd * ldf<T>(nw, i) + ldf<T>(nb, i);
      if (h32) h32[base + i] = h;
      if (hc) stf<T>(hc, base + i, h);
    }
  }
}

// One workgroup per token. The workgroup of a row's FIRST token also serves the row's next taps - 2 tokens (all those
// whose history reaches into the state slot) and then rewrites the slot, so nobody else reads or writes that slot.
// TI: type of the inputs (rows h_stride apart). ACT = false: out = h + conv(h); true: out = silu(conv(h) + bias).
template <typename TI, typename T, bool ACT>
__global__ void __launch_bounds__(256) causal_conv_kernel(const TI* __restrict__ h, int64_t h_stride,
                                                          const T* __restrict__ w, const T* __restrict__ bias,
                                                          float* __restrict__ state, const int* __restrict__ cu_q,
                                                          const int* __restrict__ first_pos,
                                                          const int* __restrict__ state_slots, T* __restrict__ out,
                                                          int B, int W, int taps) {
  const int t = blockIdx.x, K = taps - 1, c = blockIdx.y * 256 + threadIdx.x;  // one channel per thread
  const int b = row_of(cu_q, B, t);
  const int q0 = cu_q[b], n = cu_q[b + 1] - q0, off = t - q0;
  if (off >= n) return;  // a token no row owns
  const int slot = state_slots[b];
  auto put = [&](int tok, float self, float conv) {
    float a;
    if (ACT) {
      a = conv + (bias ? ldf<T>(bias, c) : 0.f);
      a /= 1.f + expf(-a);
    } else {
      a = self + conv;
    }
    stf<T>(out, (size_t)tok * W + c, a);
  };
  if (slot < 0) {  // padding row: its values go nowhere, they only have to be finite
    if (c < W) put(t, ldf<TI>(h, (size_t)t * h_stride + c), 0.f);
    return;
  }
  if (off >= K) {  // the whole history is inside the row
    if (c < W) {
      float a = 0.f;
      for (int j = 0; j < taps; ++j) a += ldf<T>(w, (size_t)c * taps + j) * ldf<TI>(h, (size_t)(t - K + j) * h_stride + c);
      put(t, ldf<TI>(h, (size_t)t * h_stride + c), a);
    }
    return;
  }
  if (off > 0) return;  // served by the workgroup of the row's first token
  const int p0 = first_pos[b];
  float* sl = state + (size_t)slot * K * W;
  // input at index p relative to the row's first token (p < 0: the state slot, or zero before the sequence's start)
  auto val = [&](int p, int c) -> float {
    if (p >= 0) return ldf<TI>(h, (size_t)(q0 + p) * h_stride + c);
    return p0 + p >= 0 ? sl[(size_t)(K + p) * W + c] : 0.f;
  };
  const int m = min(K, n);
  if (c < W) {
    for (int i = 0; i < m; ++i) {
      float a = 0.f;
      for (int j = 0; j < taps; ++j) a += ldf<T>(w, (size_t)c * taps + j) * val(i - K + j, c);
      put(q0 + i, val(i, c), a);
    }
    // the slot's entry k becomes the input K - k tokens before the NEXT token; reads run ahead of the writes
    for (int k = 0; k < K; ++k) sl[(size_t)k * W + c] = val(n - K + k, c);
  }
}

// Eight consecutive elements (16-byte aligned) as floats, and back.
template <typename T> DEVINL void ld8f(const T* p, float (&v)[8]);
template <> DEVINL void ld8f<bf16_t>(const bf16_t* p, float (&v)[8]) {
  const bf16x8 x = ld8(p);
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = bf2f(x[e]);
}
template <> DEVINL void ld8f<float>(const float* p, float (&v)[8]) {
  const f32x4 a = *reinterpret_cast<const f32x4*>(p), b = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    v[e] = a[e];
    v[4 + e] = b[e];
  }
}
template <typename T> DEVINL void st8f(T* p, const float (&v)[8]);
template <> DEVINL void st8f<bf16_t>(bf16_t* p, const float (&v)[8]) {
  bf16x8 x;
#pragma unroll
  for (int e = 0; e < 8; ++e) x[e] = f2bf(v[e]);
  st8(p, x);
}
template <> DEVINL void st8f<float>(float* p, const float (&v)[8]) {
  *reinterpret_cast<f32x4*>(p) = (f32x4){v[0], v[1], v[2], v[3]};
  *reinterpret_cast<f32x4*>(p + 4) = (f32x4){v[4], v[5], v[6], v[7]};
}

// The tokens [lo, hi) that the workgroup of tile [t0, t0 + R) of the packed batch serves when a convolution with K tokens of
// history runs along the rows: those of the tile, but a row's first K tokens - whose history reaches into the row's state
// slot - all belong to the tile of the row's first token, so that the slot has one reader. That workgroup rewrites the slot.
// single: every row has exactly one token (nothing to search for).
DEVINL void conv_span(const int* __restrict__ cu_q, int B, int T, int t0, int R, int K, bool single, int& lo, int& hi,
                      int& row) {
  if (single) {
    row = lo = t0;
    hi = min(t0 + R, T);
    return;
  }
  row = row_of(cu_q, B, t0);
  lo = t0;
  hi = min(t0 + R, min(T, cu_q[B]));
  const int q0 = cu_q[row];
  if (t0 > q0 && t0 - q0 < K) lo = min(q0 + K, cu_q[row + 1]);  // those are another tile's
  if (hi > lo) {
    const int last = row_of(cu_q, B, hi - 1), s0 = cu_q[last];
    if (s0 >= t0 && hi - s0 < K) hi = min(s0 + K, cu_q[last + 1]);
  }
}

// w[c + e][j] of eight channels and all taps: 8 (K + 1) consecutive numbers, 16-byte aligned
template <typename T, int K>
DEVINL void load_taps(const T* w, int c, float (&cw)[K + 1][8]) {
#pragma unroll
  for (int i = 0; i <= K; ++i) {
    float v[8];
    ld8f<T>(w + (size_t)c * (K + 1) + 8 * i, v);
#pragma unroll
    for (int e = 0; e < 8; ++e) cw[(8 * i + e) % (K + 1)][(8 * i + e) / (K + 1)] = v[e];
  }
}

// silu(conv(h) + bias) of rows in the storage type: eight channels a thread, R tokens a workgroup, the history in registers.
// (Rows of a multiple of 8 channels, 16-byte aligned; the fallback is causal_conv_kernel.)
template <typename T, int K>
__global__ void __launch_bounds__(256) conv_silu_vec_kernel(const T* __restrict__ h, int64_t h_stride,
                                                            const T* __restrict__ w, const T* __restrict__ bias,
                                                            float* __restrict__ state, const int* __restrict__ cu_q,
                                                            const int* __restrict__ first_pos,
                                                            const int* __restrict__ state_slots, T* __restrict__ out,
                                                            int B, int Tn, int W, int R, int single) {
  const int c = 8 * (blockIdx.y * 256 + threadIdx.x);
  int lo, hi, b;
  conv_span(cu_q, B, Tn, blockIdx.x * R, R, K, single, lo, hi, b);
  if (lo >= hi || c >= W) return;
  float cw[K + 1][8], bb[8], ring[K + 1][8];
  load_taps<T, K>(w, c, cw);
#pragma unroll
  for (int e = 0; e < 8; ++e) bb[e] = bias ? ldf<T>(bias, c + e) : 0.f;
  bool fresh_row = true;  // the ring has to be filled for the token at hand
  for (int t = lo; t < hi; ++t) {
    while (t >= cu_q[b + 1]) {
      ++b;
      fresh_row = true;
    }
    const int q0 = cu_q[b], q1 = cu_q[b + 1], slot = state_slots[b];
    float* sl = state + (size_t)max(slot, 0) * K * W + c;
    if (fresh_row) {
      fresh_row = false;
#pragma unroll
      for (int j = 0; j < K; ++j) {
        const int p = t - K + j;  // t is the row's first token, or at least K tokens into it
        if (p >= q0) ld8f<T>(h + (size_t)p * h_stride + c, ring[j]);
        else if (slot >= 0 && first_pos[b] + p - q0 >= 0) ld8f<float>(sl + (size_t)(K + p - q0) * W, ring[j]);
        else
#pragma unroll
          for (int e = 0; e < 8; ++e) ring[j][e] = 0.f;
      }
    }
    ld8f<T>(h + (size_t)t * h_stride + c, ring[K]);
    float o[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      float a = bb[e];
#pragma unroll
      for (int j = 0; j <= K; ++j) a += cw[j][e] * ring[j][e];
      o[e] = a / (1.f + expf(-a));
    }
    st8f<T>(out + (size_t)t * W + c, o);
    if (K > 0 && t == max(lo, q0) && q0 >= lo && slot >= 0) {
      // the slot's entry k becomes the input K - k tokens before the next step's first one; entries behind it are read first
      const int n = q1 - q0;
#pragma unroll
      for (int k = 0; k < K; ++k) {
        const int p = n - K + k;
        float v[8];
        if (p >= 0) {
          ld8f<T>(h + (size_t)(q0 + p) * h_stride + c, v);
        } else {
#pragma unroll
          for (int j = 0; j < K; ++j)
            if (j == K + p) {
#pragma unroll
              for (int e = 0; e < 8; ++e) v[e] = ring[j][e];
            }
        }
        st8f<float>(sl + (size_t)k * W, v);
      }
    }
#pragma unroll
    for (int j = 0; j < K; ++j)
#pragma unroll
      for (int e = 0; e < 8; ++e) ring[j][e] = ring[j + 1][e];
  }
}

// Closes a sublayer of a stream that the next sublayer reads through a convolution:
//   xo = x + LN(y; w, b);   hc = xo + conv(xo)
// One workgroup serves R consecutive tokens one after the other, eight channels a thread, the last K sums in registers; a
// tile that starts inside a row forms the K sums ahead of it once more. x and xo are different buffers. SLAB: y is the sum of
// n_slab fp32 slabs [Tn, W] (partial products of a split GEMM). hc null: only xo (K = 0, cw null).
template <typename T, int K, int MAXT, bool SLAB>
__global__ void __launch_bounds__(MAXT) norm_add_conv_kernel(
    const float* __restrict__ x, const void* __restrict__ y_, int n_slab, const T* __restrict__ w, const T* __restrict__ bias,
    const T* __restrict__ cw_, float* __restrict__ state, const int* __restrict__ cu_q, const int* __restrict__ first_pos,
    const int* __restrict__ state_slots, float* __restrict__ xo, T* __restrict__ hc, int B, int Tn, int W, int R,
    int single, float eps) {
  __shared__ float red[2][16][2];
  const int tid = threadIdx.x, wid = tid >> 6, nw = blockDim.x >> 6, c = 8 * tid;
  const bool has = c < W;
  int lo, hi, b;
  conv_span(cu_q, B, Tn, blockIdx.x * R, R, K, single, lo, hi, b);
  if (lo >= hi) return;
  float lw[8], lb[8], cw[K + 1][8], ring[K + 1][8], cx[8], cy[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) lw[e] = lb[e] = cx[e] = cy[e] = 0.f;
#pragma unroll
  for (int j = 0; j <= K; ++j)
#pragma unroll
    for (int e = 0; e < 8; ++e) cw[j][e] = ring[j][e] = 0.f;
  if (has) {
    if (cw_) load_taps<T, K>(cw_, c, cw);
    ld8f<T>(w + c, lw);
    ld8f<T>(bias + c, lb);
  }
  // numbers in wave i of a row: 512 but for the last wave that has any
  auto count = [&](int i) { return (float)max(0, min(512, W - 512 * i)); };
  const float mine = count(wid);
  auto fetch = [&](int t) {
    if (has) {
      ld8f<float>(x + (size_t)t * W + c, cx);
      if (SLAB) {
        const float* y = reinterpret_cast<const float*>(y_) + (size_t)t * W + c;
        ld8f<float>(y, cy);
#pragma unroll 4
        for (int s = 1; s < n_slab; ++s) {
          float v[8];
          ld8f<float>(y + (size_t)s * Tn * W, v);
#pragma unroll
          for (int e = 0; e < 8; ++e) cy[e] += v[e];
        }
      } else {
        ld8f<T>(reinterpret_cast<const T*>(y_) + (size_t)t * W + c, cy);
      }
    }
  };
  int parity = 0;
  // ring[K] <- the sum of the token last fetched; `next` (>= 0) is fetched meanwhile
  auto close = [&](int next) {
    float s = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) s += cy[e];
    const float mw = mine > 0.f ? wave_sum(s) / mine : 0.f;
    float m2 = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) m2 += has ? (cy[e] - mw) * (cy[e] - mw) : 0.f;
    m2 = wave_sum(m2);
    if ((tid & 63) == 0) {
      red[parity][wid][0] = mw;
      red[parity][wid][1] = m2;
    }
    float px[8], py[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      px[e] = cx[e];
      py[e] = cy[e];
    }
    if (next >= 0) fetch(next);
    __syncthreads();
    float mean = 0.f, var = 0.f;
    for (int i = 0; i < nw; ++i) mean += red[parity][i][0] * count(i);
    mean /= (float)W;
    for (int i = 0; i < nw; ++i) {
      const float d = red[parity][i][0] - mean;
      var += red[parity][i][1] + count(i) * d * d;
    }
    parity ^= 1;
    const float rstd = 1.f / sqrtf(var / (float)W + eps);
#pragma unroll
    for (int e = 0; e < 8; ++e) ring[K][e] = px[e] + ((py[e] - mean) * rstd * lw[e] + lb[e]);
  };
  auto shift = [&]() {
#pragma unroll
    for (int j = 0; j < K; ++j)
#pragma unroll
      for (int e = 0; e < 8; ++e) ring[j][e] = ring[j + 1][e];
  };
  if (lo > cu_q[b] && lo < cu_q[b + 1]) {  // inside a row (at least K tokens): the sums ahead of the tile
    if (K > 0) fetch(lo - K);
    for (int k = 0; k < K; ++k) {
      close(lo - K + k + 1);
      shift();
    }
    if (K == 0) fetch(lo);
  } else {
    fetch(lo);
  }
  for (int t = lo; t < hi; ++t) {
    while (t >= cu_q[b + 1]) ++b;
    const int q0 = cu_q[b], q1 = cu_q[b + 1], slot = state_slots[b];
    float* sl = state + (size_t)max(slot, 0) * K * W + c;
    if (t == q0) {
#pragma unroll
      for (int j = 0; j < K; ++j) {
        if (has && slot >= 0 && first_pos[b] + j - K >= 0) ld8f<float>(sl + (size_t)j * W, ring[j]);
        else
#pragma unroll
          for (int e = 0; e < 8; ++e) ring[j][e] = 0.f;
      }
    }
    close(t + 1 < hi ? t + 1 : -1);
    float o[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      float a = 0.f;
#pragma unroll
      for (int j = 0; j <= K; ++j) a += cw[j][e] * ring[j][e];
      o[e] = slot >= 0 ? ring[K][e] + a : ring[K][e];
    }
    if (has) {
      st8f<float>(xo + (size_t)t * W + c, ring[K]);
      if (hc) st8f<T>(hc + (size_t)t * W + c, o);
    }
    shift();
    if (K > 0 && q0 >= lo && slot >= 0) {  // this workgroup served the row's first token: it leaves the row's last K sums
      if (t == hi - 1 && q1 > hi) {
        for (int u = max(hi, q1 - K); u < q1; ++u) {
          fetch(u);
          close(-1);
          shift();
        }
      }
      if ((t == q1 - 1 || t == hi - 1) && has) {
#pragma unroll
        for (int j = 0; j < K; ++j) st8f<float>(sl + (size_t)j * W, ring[j]);
      }
    }
  }
}

template <typename T>
__global__ void __launch_bounds__(1024) embed_bigram_norm_kernel(
    const int64_t* __restrict__ tokens, const T* __restrict__ embed, const T* __restrict__ bigram, int buckets,
    int64_t mul_prev, int64_t mul_cur, const T* __restrict__ w, const T* __restrict__ bias, float eps,
    const int* __restrict__ cu_q, const int* __restrict__ first_pos, const int* __restrict__ state_slots,
    int* __restrict__ prev_state, float* __restrict__ out, int B, int W, int vocab) {
  extern __shared__ float row[];
  float* red = row + W;
  __shared__ int64_t big_row;
  const int t = blockIdx.x;
  int64_t tok = tokens[t];
  tok = tok < 0 ? 0 : (tok >= vocab ? vocab - 1 : tok);
  if (threadIdx.x == 0) {
    int64_t r = -1;
    if (bigram) {
      const int b = row_of(cu_q, B, t);
      const int q0 = cu_q[b], n = cu_q[b + 1] - q0, off = t - q0, slot = state_slots[b];
      if (off < n && slot >= 0) {
        if (first_pos[b] + off == 0) {
          r = buckets;
        } else {
          const int64_t prev = off > 0 ? tokens[t - 1] : (int64_t)prev_state[slot];
          r = (prev * mul_prev + tok * mul_cur) % (int64_t)buckets;
          if (r < 0) r += buckets;
        }
        // the row's first token owns the slot: it has read the token before, now it leaves the row's last one
        if (off == 0) prev_state[slot] = (int)tokens[q0 + n - 1];
      }
    }
    big_row = r;
  }
  __syncthreads();
  const int64_t r = big_row;
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    float v = ldf<T>(embed, (size_t)tok * W + i);
    if (r >= 0) v += ldf<T>(bigram, (size_t)r * W + i);
    row[i] = v;
  }
  __syncthreads();
  float mean, rstd;
  row_stats(row, W, eps, red, mean, rstd);
  for (int i = threadIdx.x; i < W; i += blockDim.x)
    out[(size_t)t * W + i] = (row[i] - mean) * rstd * ldf<T>(w, i) + ldf<T>(bias, i);
}

}  // namespace

// Threads of a one-token workgroup: a few elements per thread, so that a launch of few tokens (a decode step) is not a
// chain of dependent loads.
static int row_threads(int W) { return W > 2048 ? 1024 : (W > 512 ? 512 : 256); }

static int row_lds(int W, size_t* bytes) {
  *bytes = (size_t)(W + 16) * sizeof(float);
  return *bytes <= 64 * 1024 ? 0 : -2;  // rows up to 16368 channels
}

// Threads of a one-token workgroup in the vector variants: four elements a thread and pass where the row allows.
static int row_threads4(int W) {
  const int t = ((W / 4 + 63) / 64) * 64;
  return t > 1024 ? 1024 : (t < 64 ? 64 : t);
}
static bool aligned16(const void* p) { return ((uintptr_t)p & 15) == 0; }

extern "C" int areal_layer_norm32(const float* x, const void* w, const void* b, float* o32, void* oc, int T, int W,
                                  float eps, int dt, hipStream_t st) {
  if (T == 0) return 0;
  size_t lds;
  if (W <= 0 || row_lds(W, &lds)) return -2;
  const bool v4 = W % 4 == 0 && aligned16(x) && aligned16(w) && aligned16(b) && aligned16(o32) && aligned16(oc);
#define LN_LAUNCH(TT, V4, NTHR)                                                                               \
  hipLaunchKernelGGL((layer_norm32_kernel<TT, V4>), dim3(T), dim3(NTHR), lds, st, x, (const TT*)w, (const TT*)b, \
                     o32, (TT*)(dt == 0 ? oc : nullptr), W, eps)
  if (dt == 0) {
    if (v4) LN_LAUNCH(bf16_t, true, row_threads4(W));
    else LN_LAUNCH(bf16_t, false, row_threads(W));
  } else {
    if (v4) LN_LAUNCH(float, true, row_threads4(W));
    else LN_LAUNCH(float, false, row_threads(W));
  }
#undef LN_LAUNCH
  return (int)hipGetLastError();
}

extern "C" int areal_gated_norm_add(float* x, const void* y, const void* gate, const void* w, const void* b,
                                    const void* scale, const void* nw, const void* nb, float* h32, void* hc, int T,
                                    int W, float eps, int dt, hipStream_t st) {
  if (T == 0) return 0;
  size_t lds;
  if (W <= 0 || row_lds(W, &lds)) return -2;
  const bool v4 = W % 4 == 0 && aligned16(x) && aligned16(y) && aligned16(gate) && aligned16(w) && aligned16(b) &&
                  aligned16(scale) && aligned16(nw) && aligned16(nb) && aligned16(h32) && aligned16(hc);
#define GN_LAUNCH(TT, V4, NTHR)                                                                                  \
  hipLaunchKernelGGL((gated_norm_add_kernel<TT, V4>), dim3(T), dim3(NTHR), lds, st, x, (const TT*)y,             \
                     (const TT*)gate, (const TT*)w, (const TT*)b, (const TT*)scale, (const TT*)nw, (const TT*)nb, \
                     h32, (TT*)(dt == 0 ? hc : nullptr), W, eps)
  if (dt == 0) {
    if (v4) GN_LAUNCH(bf16_t, true, row_threads4(W));
    else GN_LAUNCH(bf16_t, false, row_threads(W));
  } else {
    if (v4) GN_LAUNCH(float, true, row_threads4(W));
    else GN_LAUNCH(float, false, row_threads(W));
  }
#undef GN_LAUNCH
  return (int)hipGetLastError();
}

extern "C" int areal_canon_conv(const float* h, const void* w, float* state, const int* cu_q, const int* first_pos,
                                const int* state_slots, void* out, int B, int T, int W, int taps, int dt,
                                hipStream_t st) {
  if (T == 0 || B == 0) return 0;
  if (taps < 1 || (taps > 1 && !state) || (W + 255) / 256 > 65535) return -1;
  const dim3 grid(T, (W + 255) / 256);
  if (dt == 0)
    hipLaunchKernelGGL((causal_conv_kernel<float, bf16_t, false>), grid, dim3(256), 0, st, h, (int64_t)W, (const bf16_t*)w,
                       (const bf16_t*)nullptr, state, cu_q, first_pos, state_slots, (bf16_t*)out, B, W, taps);
  else
    hipLaunchKernelGGL((causal_conv_kernel<float, float, false>), grid, dim3(256), 0, st, h, (int64_t)W, (const float*)w,
                       (const float*)nullptr, state, cu_q, first_pos, state_slots, (float*)out, B, W, taps);
  return (int)hipGetLastError();
}

// out [T, W] = silu(conv(h) + bias), h rows in the storage type, h_stride apart; bias [W] or null
extern "C" int areal_conv_silu(const void* h, int64_t h_stride, const void* w, const void* bias, float* state,
                               const int* cu_q, const int* first_pos, const int* state_slots, void* out, int B, int T,
                               int W, int taps, int max_q, int dt, hipStream_t st) {
  if (T == 0 || B == 0) return 0;
  if (taps < 1 || (taps > 1 && !state) || (W + 255) / 256 > 65535) return -1;
  const int single = max_q == 1 && T == B;
  const int R = T <= 512 ? 1 : 16;
  if (taps <= 4 && W % 8 == 0 && h_stride % 8 == 0 && aligned16(h) && aligned16(w) && aligned16(out) &&
      aligned16(state)) {
    const dim3 vgrid((T + R - 1) / R, (W / 8 + 255) / 256);
#define CONV(TT, KV)                                                                                                \
  hipLaunchKernelGGL((conv_silu_vec_kernel<TT, KV>), vgrid, dim3(256), 0, st, (const TT*)h, h_stride, (const TT*)w, \
                     (const TT*)bias, state, cu_q, first_pos, state_slots, (TT*)out, B, T, W, R, single)
#define CONV_K(TT)                  \
  do {                              \
    if (taps == 1) CONV(TT, 0);     \
    else if (taps == 2) CONV(TT, 1); \
    else if (taps == 3) CONV(TT, 2); \
    else CONV(TT, 3);               \
  } while (0)
    if (dt == 0) CONV_K(bf16_t);
    else CONV_K(float);
#undef CONV_K
#undef CONV
    return (int)hipGetLastError();
  }
  const dim3 grid(T, (W + 255) / 256);
  if (dt == 0)
    hipLaunchKernelGGL((causal_conv_kernel<bf16_t, bf16_t, true>), grid, dim3(256), 0, st, (const bf16_t*)h, h_stride,
                       (const bf16_t*)w, (const bf16_t*)bias, state, cu_q, first_pos, state_slots, (bf16_t*)out, B, W, taps);
  else
    hipLaunchKernelGGL((causal_conv_kernel<float, float, true>), grid, dim3(256), 0, st, (const float*)h, h_stride,
                       (const float*)w, (const float*)bias, state, cu_q, first_pos, state_slots, (float*)out, B, W, taps);
  return (int)hipGetLastError();
}

// Whether areal_norm_add_conv serves rows of W channels and this many taps (0: no convolution).
extern "C" int areal_norm_add_conv_serves(int W, int taps) { return taps >= 0 && taps <= 4 && W > 0 && W % 8 == 0 && W <= 8192; }

// xo = x + LN(y; w, b) and, with taps > 0, hc = xo + conv(xo) (conv weights cw [W, taps], state as in areal_canon_conv); x, xo
// fp32 in different buffers; every pointer 16-byte aligned. n_slab > 0: y is the sum of n_slab fp32 slabs [T, W] that follow
// each other; 0: one row per token in the storage type. max_q: longest row.
extern "C" int areal_norm_add_conv(const float* x, const void* y, int n_slab, const void* w, const void* b, const void* cw,
                                   float* state, const int* cu_q, const int* first_pos, const int* state_slots, float* xo,
                                   void* hc, int B, int T, int W, int taps, int max_q, float eps, int dt, hipStream_t st) {
  if (T == 0 || B == 0) return 0;
  if (!areal_norm_add_conv_serves(W, taps) || (taps > 1 && !state) || x == xo || (taps > 0) != (hc != nullptr)) return -1;
  if (!aligned16(x) || !aligned16(y) || !aligned16(w) || !aligned16(b) || !aligned16(cw) || !aligned16(state) ||
      !aligned16(xo) || !aligned16(hc))
    return -2;
  const int R = T <= 512 ? 1 : 16, nthr = ((W / 8 + 63) / 64) * 64, single = max_q == 1 && T == B;
#define CLOSE_S(TT, KV, MT, SL)                                                                                     \
  hipLaunchKernelGGL((norm_add_conv_kernel<TT, KV, MT, SL>), dim3((T + R - 1) / R), dim3(nthr), 0, st, x, y, n_slab,  \
                     (const TT*)w, (const TT*)b, (const TT*)cw, state, cu_q, first_pos, state_slots, xo, (TT*)hc, B,  \
                     T, W, R, single, eps)
#define CLOSE(TT, KV)                                      \
  do {                                                     \
    if (nthr <= 512) {                                     \
      if (n_slab > 0) CLOSE_S(TT, KV, 512, true);          \
      else CLOSE_S(TT, KV, 512, false);                    \
    } else {                                               \
      if (n_slab > 0) CLOSE_S(TT, KV, 1024, true);         \
      else CLOSE_S(TT, KV, 1024, false);                   \
    }                                                      \
  } while (0)
#define CLOSE_K(TT)                   \
  do {                                \
    if (taps <= 1) CLOSE(TT, 0);      \
    else if (taps == 2) CLOSE(TT, 1); \
    else if (taps == 3) CLOSE(TT, 2); \
    else CLOSE(TT, 3);                \
  } while (0)
  if (dt == 0) CLOSE_K(bf16_t);
  else CLOSE_K(float);
#undef CLOSE_K
#undef CLOSE
#undef CLOSE_S
  return (int)hipGetLastError();
}

extern "C" int areal_embed_bigram_norm(const int64_t* tokens, const void* embed, const void* bigram, int buckets,
                                       int64_t mul_prev, int64_t mul_cur, const void* w, const void* bias, float eps,
                                       const int* cu_q, const int* first_pos, const int* state_slots, int* prev_state,
                                       float* out, int B, int T, int W, int vocab, int dt, hipStream_t st) {
  if (T == 0 || B == 0) return 0;
  size_t lds;
  if (W <= 0 || row_lds(W, &lds)) return -2;
  if (bigram && (buckets < 1 || !prev_state)) return -1;
  if (dt == 0)
    hipLaunchKernelGGL(embed_bigram_norm_kernel<bf16_t>, dim3(T), dim3(row_threads(W)), lds, st, tokens, (const bf16_t*)embed,
                       (const bf16_t*)bigram, buckets, mul_prev, mul_cur, (const bf16_t*)w, (const bf16_t*)bias, eps,
                       cu_q, first_pos, state_slots, prev_state, out, B, W, vocab);
  else
    hipLaunchKernelGGL(embed_bigram_norm_kernel<float>, dim3(T), dim3(row_threads(W)), lds, st, tokens, (const float*)embed,
                       (const float*)bigram, buckets, mul_prev, mul_cur, (const float*)w, (const float*)bias, eps,
                       cu_q, first_pos, state_slots, prev_state, out, B, W, vocab);
  return (int)hipGetLastError();
}
