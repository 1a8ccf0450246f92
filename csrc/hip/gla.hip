// Gated linear attention: a matrix state per head whose rows (one per key channel) decay by a data-dependent factor.
//
//   alpha_t = sigmoid(z_t)^(1 / tau) = exp(-softplus(-z_t) / tau)        z_t: one logit per head and key channel
//   S_t     = diag(alpha_t) S_(t-1) + k_t v_t^T      [D, V]              o_t = S_t^T (q_t * q_scale)
//   y_t     = o_t / rms(o_t over V) * w * silu(g_t)                      per head; w [V] is shared by the heads; `sigmoid`:
//                                                                        times sigmoid(g_t) instead
//
// q, k, v and g are columns of one projection (storage type T); z arrives as fp32 logits (plus a bias in T), and the
// decays, the state, the read-out and the norm are fp32. State slots [slots, heads, D, V] live in device memory
// between steps: a row whose first token has position 0 starts from S = 0 whatever its slot held before; a row with a
// negative slot is skipped (its outputs are zero).
//
// `gla_scan_kernel`: token by token, one workgroup of four waves per (row, head, 64 value columns); wave r keeps a
// quarter of the rows of S in registers (lane c: column c). Keys, queries and decays of 8 tokens are staged ahead.
// `gla_chunk_kernel`: prompt portions in chunks of 16 tokens. With b_t = sum_{u <= t} ln alpha_u (per channel, from the
// chunk's start; every b <= 0):
//
//   o_t   = (q_t * exp(b_t))^T S_prev + sum_{s <= t} A[t, s] v_s,     A[t, s] = sum_d q_t[d] k_s[d] exp(b_t[d] - b_s[d])
//   S_new = diag(exp(b_L)) S_prev + sum_s (k_s * exp(b_L - b_s)) v_s^T
//
// Every exponent is <= 0: nothing overflows whatever the decays are, and nothing is divided.
// `gla_out_kernel`: per-head RMS norm of the read-out, weight, SiLU gate.
#include "common.hpp"

namespace {

template <typename T> DEVINL float ldf(const T* p, size_t i);
template <> DEVINL float ldf<bf16_t>(const bf16_t* p, size_t i) { return bf2f(p[i]); }
template <> DEVINL float ldf<float>(const float* p, size_t i) { return p[i]; }
template <typename T> DEVINL void stf(T* p, size_t i, float v);
template <> DEVINL void stf<bf16_t>(bf16_t* p, size_t i, float v) { p[i] = f2bf(v); }
template <> DEVINL void stf<float>(float* p, size_t i, float v) { p[i] = v; }

// ln sigmoid(z) / tau; bf16 storage: hardware exponential and logarithm (a short series where 1 + e would lose e's digits)
template <typename T> DEVINL float log_decay(float z, float inv_tau) {
  if (sizeof(T) == 2) {
    const float e = __expf(-fabsf(z));
    const float l = e < 0.0156f ? e * (1.f - e * (0.5f - 0.33333333f * e)) : __logf(1.f + e);
    return -(fmaxf(-z, 0.f) + l) * inv_tau;
  }
  return -(fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z)))) * inv_tau;
}

constexpr int TC = 8;  // tokens staged per step of the loop
constexpr int RW = 4;  // waves of a workgroup

template <typename T, int DP>
__global__ void __launch_bounds__(64 * RW) gla_scan_kernel(
    const T* __restrict__ proj, int64_t row_stride, int q_off, int k_off, int v_off, const float* __restrict__ z,
    int64_t z_stride, const T* __restrict__ z_bias, float inv_tau, float q_scale, const int* __restrict__ cu_q,
    const int* __restrict__ first_pos, const int* __restrict__ state_slots, float* __restrict__ S,
    float* __restrict__ obuf, int NH, int D, int V) {
  constexpr int DQ = DP / RW;
  __shared__ float kqa[TC][3][DP];
  __shared__ float hpart[RW][TC][64];
  const int b = blockIdx.x, hd = blockIdx.y, tid = threadIdx.x, lane = tid & 63, r = tid >> 6;
  const int col = blockIdx.z * 64 + lane;
  const bool has = col < V;
  const int slot = state_slots[b];
  const int t_lo = cu_q[b], t_hi = cu_q[b + 1];
  if (slot < 0) {
    if (r == 0)
      for (int t = t_lo; t < t_hi; ++t)
        if (has) obuf[((size_t)t * NH + hd) * V + col] = 0.f;
    return;
  }
  if (t_hi <= t_lo) return;
  const bool fresh = first_pos[b] == 0;
  const size_t sbase = ((size_t)slot * NH + hd) * D;
  const int d0 = r * DQ;
  float s[DQ];
#pragma unroll
  for (int d = 0; d < DQ; ++d) s[d] = (!fresh && has && d0 + d < D) ? S[(sbase + d0 + d) * V + col] : 0.f;
  for (int tb = t_lo; tb < t_hi; tb += TC) {
    const int nt = min(TC, t_hi - tb);
    __syncthreads();  // the step before is finished with the staged operands and the partials
    for (int i = tid; i < TC * DP; i += 64 * RW) {
      const int d = i % DP, tt = i / DP;
      const bool live = tt < nt && d < D;
      const size_t tok = (size_t)(tb + min(tt, nt - 1));
      const T* row = proj + tok * row_stride;
      kqa[tt][0][d] = live ? ldf<T>(row, k_off + hd * D + d) : 0.f;
      kqa[tt][1][d] = live ? ldf<T>(row, q_off + hd * D + d) * q_scale : 0.f;
      kqa[tt][2][d] = live ? expf(log_decay<T>(z[tok * z_stride + hd * D + d] + (z_bias ? ldf<T>(z_bias, hd * D + d) : 0.f),
                                            inv_tau))
                           : 1.f;
    }
    float vv[TC];
#pragma unroll
    for (int tt = 0; tt < TC; ++tt)
      vv[tt] = (tt < nt && has) ? ldf<T>(proj + (size_t)(tb + tt) * row_stride, v_off + hd * V + col) : 0.f;
    __syncthreads();
#pragma unroll
    for (int tt = 0; tt < TC; ++tt) {
      if (tt < nt) {
        float hacc = 0.f;
#pragma unroll
        for (int d = 0; d < DQ; ++d) {
          s[d] = kqa[tt][2][d0 + d] * s[d] + vv[tt] * kqa[tt][0][d0 + d];
          hacc += s[d] * kqa[tt][1][d0 + d];
        }
        hpart[r][tt][lane] = hacc;
      }
    }
    __syncthreads();
#pragma unroll
    for (int tt = 0; tt < TC; ++tt) {
      if (tt < nt && (tt % RW) == r && has) {
        float hsum = 0.f;
#pragma unroll
        for (int w = 0; w < RW; ++w) hsum += hpart[w][tt][lane];
        obuf[((size_t)(tb + tt) * NH + hd) * V + col] = hsum;
      }
    }
  }
  if (has) {
#pragma unroll
    for (int d = 0; d < DQ; ++d)
      if (d0 + d < D) S[(sbase + d0 + d) * V + col] = s[d];
  }
}

// Prompt portions: chunks of CT tokens, in two launches. Whatever does not depend on the state is formed for all
// chunks at once by `gla_prep_kernel` (one workgroup per (chunk, row, head), thousands of them): the per-channel log
// decays summed along the chunk's tokens (b_t), q_t * exp(b_t), k_s * exp(b_L - b_s), exp(b_L), and the lower triangle
// A[t, s] = sum_d q_t[d] k_s[d] exp(b_t[d] - b_s[d]), pair by pair so that every exponent is <= 0. It leaves them in the
// order in which `gla_chunk_kernel` reads them as matrix-core operands, padded with zeros to CT tokens and DP channels:
// per (chunk slot, head) q~ [CT][DP], k~^T [DP][CT], exp(b_L) [DP], A [CT][CT]. `gla_chunk_kernel` then walks a row's chunks
// with nothing but products on the fp32 matrix cores (MFMA 16x16x4): a wave owns 16 value columns and keeps its slice of the
// state in registers, which are at once the B operand of the read-out q~ S_prev + A V and the accumulator of the move to
// the chunk's end diag(exp(b_L)) S_prev + k~^T V (lane: column, channels 16 i + 4 quad .. + 3). Waves share nothing: no LDS,
// no barriers; the operands of the next two chunks are fetched under the matrix work.
constexpr int CT = 16;

// Slot of the chunk that starts at token tb of row b (first token t_lo) in the scratch buffers; T / CT + B + 1 slots.
DEVINL size_t chunk_slot(int t_lo, int tb, int b) { return (size_t)(t_lo / CT + b + (tb - t_lo) / CT); }
template <int DP> constexpr size_t chunk_floats() { return 2 * CT * DP + DP + CT * CT; }

// bf16 storage: v_exp_f32 (relative error ~1e-6, far below the storage's); fp32 storage: the library's exp
template <typename T> DEVINL float exp_le0(float x) { return sizeof(T) == 2 ? __expf(x) : expf(x); }

template <typename T, int DP>
__global__ void __launch_bounds__(256) gla_prep_kernel(
    const T* __restrict__ proj, int64_t row_stride, int q_off, int k_off, const float* __restrict__ z, int64_t z_stride,
    const T* __restrict__ z_bias, float inv_tau, float q_scale, const int* __restrict__ cu_q,
    const int* __restrict__ state_slots, float* __restrict__ scratch, int NH, int D) {
  constexpr int QS = DP + 1;  // odd stride: the pair loop's 16 key rows fall on different banks
  __shared__ float Qr[CT * QS], Kr[CT * QS], Bs[CT * QS];
  const int b = blockIdx.y, hd = blockIdx.z, tid = threadIdx.x;
  const int t_lo = cu_q[b], t_hi = cu_q[b + 1], tb = t_lo + CT * blockIdx.x;
  if (tb >= t_hi || state_slots[b] < 0) return;
  const int nt = min(CT, t_hi - tb);
  for (int i = tid; i < CT * DP; i += 256) {
    const int d = i % DP, tt = i / DP;
    const bool live = tt < nt && d < D;
    const size_t tok = (size_t)(tb + min(tt, nt - 1));
    const T* row = proj + tok * row_stride;
    const int dc = min(d, D - 1);
    Kr[tt * QS + d] = live ? ldf<T>(row, k_off + hd * D + dc) : 0.f;
    Qr[tt * QS + d] = live ? ldf<T>(row, q_off + hd * D + dc) * q_scale : 0.f;
    // rows past the chunk's end and padding channels do not decay
    Bs[tt * QS + d] = live ? log_decay<T>(z[tok * z_stride + hd * D + dc] + (z_bias ? ldf<T>(z_bias, hd * D + dc) : 0.f), inv_tau)
                           : 0.f;
  }
  __syncthreads();
  if (tid < DP) {  // running sums along the chunk's tokens, one channel a thread
    float run = 0.f;
#pragma unroll
    for (int tt = 0; tt < CT; ++tt) {
      run += Bs[tt * QS + tid];
      Bs[tt * QS + tid] = run;
    }
  }
  __syncthreads();
  float* qd = scratch + (chunk_slot(t_lo, tb, b) * NH + hd) * chunk_floats<DP>();
  float *kd = qd + CT * DP, *el = kd + CT * DP, *abuf = el + DP;
  for (int i = tid; i < CT * DP; i += 256) {
    const int d = i % DP, tt = i / DP;
    qd[i] = Qr[tt * QS + d] * exp_le0<T>(Bs[tt * QS + d]);
    const int kt = i % CT, kc = i / CT;
    kd[i] = Kr[kt * QS + kc] * exp_le0<T>(Bs[(CT - 1) * QS + kc] - Bs[kt * QS + kc]);
  }
  for (int i = tid; i < DP; i += 256) el[i] = exp_le0<T>(Bs[(CT - 1) * QS + i]);
  {  // the chunk's own pairs: thread (t, s), s <= t
    const int t = tid / CT, sx = tid % CT;
    float a0 = 0.f, a1 = 0.f;
    if (sx <= t && t < nt) {
      const float *qt = Qr + t * QS, *ks = Kr + sx * QS, *bt = Bs + t * QS, *bs = Bs + sx * QS;
#pragma unroll 4
      for (int d = 0; d < DP; d += 2) {
        a0 += qt[d] * ks[d] * exp_le0<T>(bt[d] - bs[d]);
        a1 += qt[d + 1] * ks[d + 1] * exp_le0<T>(bt[d + 1] - bs[d + 1]);
      }
    }
    abuf[tid] = a0 + a1;
  }
}

template <typename T, int DP>
__global__ void __launch_bounds__(256) gla_chunk_kernel(
    const float* __restrict__ scratch, const T* __restrict__ proj, int64_t row_stride, int v_off,
    const int* __restrict__ cu_q, const int* __restrict__ first_pos, const int* __restrict__ state_slots,
    float* __restrict__ S, float* __restrict__ obuf, int NH, int D, int V) {
  constexpr int NB = DP / 16;  // blocks of 16 state rows
  const int b = blockIdx.x, hd = blockIdx.y, lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int r16 = lane & 15, quad = lane >> 4, c = blockIdx.z * 64 + 16 * w + r16;
  const bool has = c < V;
  const int slot = state_slots[b];
  const int t_lo = cu_q[b], t_hi = cu_q[b + 1];
  if (slot < 0) {
    for (int t = t_lo + quad; t < t_hi; t += 4)
      if (has) obuf[((size_t)t * NH + hd) * V + c] = 0.f;
    return;
  }
  if (t_hi <= t_lo || blockIdx.z * 64 + 16 * w >= V) return;
  const bool fresh = first_pos[b] == 0;
  float* Sp = S + ((size_t)slot * NH + hd) * D * V + min(c, V - 1);
  f32x4 s[NB];
#pragma unroll
  for (int rb = 0; rb < NB; ++rb)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * rb + 4 * quad + i;
      s[rb][i] = (!fresh && has && d < D) ? Sp[(size_t)d * V] : 0.f;
    }
  struct Operands {
    f32x4 q[NB], k[NB], e[NB], a;
    T v[4];  // as loaded: nothing waits for a load before its chunk's turn
  };
  const T* vp = proj + v_off + hd * V + min(c, V - 1);
  auto fetch = [&](Operands& o, int tb) {
    const float* base = scratch + (chunk_slot(t_lo, tb, b) * NH + hd) * chunk_floats<DP>();
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      o.q[i] = *reinterpret_cast<const f32x4*>(base + r16 * DP + 16 * i + 4 * quad);
      o.k[i] = *reinterpret_cast<const f32x4*>(base + CT * DP + (16 * i + r16) * CT + 4 * quad);
      o.e[i] = *reinterpret_cast<const f32x4*>(base + 2 * CT * DP + 16 * i + 4 * quad);
    }
    o.a = *reinterpret_cast<const f32x4*>(base + 2 * CT * DP + DP + r16 * CT + 4 * quad);
#pragma unroll
    for (int i = 0; i < 4; ++i)  // rows past the chunk's end meet zeros in A and k~: any finite value will do
      o.v[i] = vp[(size_t)min(tb + 4 * quad + i, t_hi - 1) * row_stride];
  };
  auto chunk = [&](const Operands& o, int tb) {
    f32x4 v;
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = (float)o.v[i];
    f32x4 acc = {0.f, 0.f, 0.f, 0.f}, acc2 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(o.q[i][0], s[i][0], acc, 0, 0, 0);
      acc2 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.q[i][1], s[i][1], acc2, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(o.q[i][2], s[i][2], acc, 0, 0, 0);
      acc2 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.q[i][3], s[i][3], acc2, 0, 0, 0);
    }
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(o.a[0], v[0], acc, 0, 0, 0);
    acc2 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.a[1], v[1], acc2, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(o.a[2], v[2], acc, 0, 0, 0);
    acc2 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.a[3], v[3], acc2, 0, 0, 0);
#pragma unroll
    for (int rb = 0; rb < NB; ++rb) s[rb] *= o.e[rb];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int rb = 0; rb < NB; ++rb) s[rb] = __builtin_amdgcn_mfma_f32_16x16x4f32(o.k[rb][i], v[i], s[rb], 0, 0, 0);
    acc += acc2;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = tb + 4 * quad + i;
      if (t < t_hi && has) obuf[((size_t)t * NH + hd) * V + c] = acc[i];
    }
  };
  // three sets of operands: a chunk's loads are under way for two chunks
  Operands o0, o1, o2;
  fetch(o0, t_lo);
  if (t_lo + CT < t_hi) fetch(o1, t_lo + CT);
  for (int tb = t_lo; tb < t_hi; tb += 3 * CT) {
    if (tb + 2 * CT < t_hi) fetch(o2, tb + 2 * CT);
    chunk(o0, tb);
    if (tb + CT >= t_hi) break;
    if (tb + 3 * CT < t_hi) fetch(o0, tb + 3 * CT);
    chunk(o1, tb + CT);
    if (tb + 2 * CT >= t_hi) break;
    if (tb + 4 * CT < t_hi) fetch(o1, tb + 4 * CT);
    chunk(o2, tb + 2 * CT);
  }
#pragma unroll
  for (int rb = 0; rb < NB; ++rb)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * rb + 4 * quad + i;
      if (has && d < D) Sp[(size_t)d * V] = s[rb][i];
    }
}

// One wave per (token, head): y = o / rms(o over V) * w * silu(gate)
template <typename T>
__global__ void __launch_bounds__(256) gla_out_kernel(const float* __restrict__ obuf, const T* __restrict__ gate,
                                                      int64_t gate_stride, const T* __restrict__ w, T* __restrict__ out,
                                                      int64_t out_stride, float out_scale, int64_t n_rows, int NH, int V,
                                                      float eps, int vec, int sigmoid) {
  const int lane = threadIdx.x & 63;
  const int64_t row = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (row >= n_rows) return;
  const int64_t t = row / NH;
  const int hd = (int)(row % NH);
  const float* o = obuf + row * V;
  if (vec) {  // rows of a multiple of 4 numbers, 8- / 16-byte aligned: four a lane and step
    float ss = 0.f;
    for (int i = 4 * lane; i < V; i += 256) {
      const f32x4 x = *reinterpret_cast<const f32x4*>(o + i);
      ss += x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
    }
    const float r = 1.f / sqrtf(wave_sum(ss) / (float)V + eps) * out_scale;
    typedef T t4 __attribute__((ext_vector_type(4)));
    for (int i = 4 * lane; i < V; i += 256) {
      const f32x4 x = *reinterpret_cast<const f32x4*>(o + i);
      const t4 g4 = *reinterpret_cast<const t4*>(gate + t * gate_stride + hd * V + i), w4 = *reinterpret_cast<const t4*>(w + i);
      t4 y;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float g = (float)g4[e];
        y[e] = (T)(x[e] * r * (float)w4[e] * ((sigmoid ? 1.f : g) / (1.f + (sizeof(T) == 2 ? __expf(-g) : expf(-g)))));
      }
      *reinterpret_cast<t4*>(out + t * out_stride + hd * V + i) = y;
    }
    return;
  }
  float ss = 0.f;
  for (int i = lane; i < V; i += 64) ss += o[i] * o[i];
  const float r = 1.f / sqrtf(wave_sum(ss) / (float)V + eps);
  for (int i = lane; i < V; i += 64) {
    const float g = ldf<T>(gate, t * gate_stride + hd * V + i);
    stf<T>(out, t * out_stride + hd * V + i, o[i] * r * ldf<T>(w, i) * ((sigmoid ? 1.f : g) / (1.f + expf(-g))) * out_scale);
  }
}

}  // namespace

// Floats of the chunked form's scratch.
extern "C" int64_t areal_gla_scratch(int T, int B, int NH, int D) {
  const size_t per = D <= 32 ? chunk_floats<32>() : (D <= 64 ? chunk_floats<64>() : chunk_floats<128>());
  return (int64_t)(T / CT + B + 1) * NH * per;
}

// proj rows hold (at q_off / k_off / v_off) NH query heads of D, NH key heads of D, NH value heads of V. z fp32 rows of
// NH D decay logits (z_stride apart), z_bias [NH D] in the storage type or null. S [slots, NH, D, V] fp32; obuf
// [T, NH, V] fp32. scratch: areal_gla_scratch floats, 16-byte aligned, for the chunked form (rows of 16 tokens and more,
// D <= 128), or null: token by token.
extern "C" int areal_gla_scan(const void* proj, int64_t row_stride, int q_off, int k_off, int v_off, const float* z,
                              int64_t z_stride, const void* z_bias, float tau, float q_scale, const int* cu_q,
                              const int* first_pos, const int* state_slots, float* S, float* obuf, float* scratch, int T,
                              int B, int NH, int D, int V, int max_q, int dt, hipStream_t st) {
  if (B == 0) return 0;
  if (D > 256 || D <= 0 || V <= 0 || !(tau > 0.f)) return -1;
  const dim3 grid(B, NH, (V + 63) / 64);
  const float inv_tau = 1.f / tau;
  if (max_q >= CT && D <= 128 && scratch) {
    const dim3 pgrid((max_q + CT - 1) / CT, B, NH);
#define CHUNK(TT, DPV)                                                                                                 \
  do {                                                                                                                 \
    hipLaunchKernelGGL((gla_prep_kernel<TT, DPV>), pgrid, dim3(256), 0, st, (const TT*)proj, row_stride, q_off, k_off,  \
                       z, z_stride, (const TT*)z_bias, inv_tau, q_scale, cu_q, state_slots, scratch, NH, D);            \
    hipLaunchKernelGGL((gla_chunk_kernel<TT, DPV>), grid, dim3(256), 0, st, scratch, (const TT*)proj, row_stride,       \
                       v_off, cu_q, first_pos, state_slots, S, obuf, NH, D, V);                                        \
  } while (0)
#define PICKC(TT)                    \
  do {                               \
    if (D <= 32) CHUNK(TT, 32);      \
    else if (D <= 64) CHUNK(TT, 64); \
    else CHUNK(TT, 128);             \
  } while (0)
    if (dt == 0) PICKC(bf16_t);
    else PICKC(float);
#undef PICKC
#undef CHUNK
    return (int)hipGetLastError();
  }
#define LAUNCH(TT, DPV)                                                                                          \
  hipLaunchKernelGGL((gla_scan_kernel<TT, DPV>), grid, dim3(64 * RW), 0, st, (const TT*)proj, row_stride, q_off,  \
                     k_off, v_off, z, z_stride, (const TT*)z_bias, inv_tau, q_scale, cu_q, first_pos, state_slots, S, \
                     obuf, NH, D, V)
#define PICK(TT)                        \
  do {                                  \
    if (D <= 32) LAUNCH(TT, 32);        \
    else if (D <= 64) LAUNCH(TT, 64);   \
    else if (D <= 128) LAUNCH(TT, 128); \
    else LAUNCH(TT, 256);               \
  } while (0)
  if (dt == 0) PICK(bf16_t);
  else PICK(float);
#undef PICK
#undef LAUNCH
  return (int)hipGetLastError();
}

// obuf [T, NH, V] fp32, gate rows of NH V with gate_stride, w [V]; out rows of NH V numbers, out_stride apart, times out_scale
extern "C" int areal_gla_out(const float* obuf, const void* gate, int64_t gate_stride, const void* w, void* out,
                             int64_t out_stride, float out_scale, int T, int NH, int V, float eps, int sigmoid,
                             int dt, hipStream_t st) {
  if (T == 0) return 0;
  const int64_t n = (int64_t)T * NH;
  const dim3 grid((unsigned)((n + 3) / 4));
  const int vec = V % 4 == 0 && gate_stride % 4 == 0 && out_stride % 4 == 0 && (uintptr_t)obuf % 16 == 0 &&
                  (((uintptr_t)gate | (uintptr_t)w | (uintptr_t)out) % (dt == 0 ? 8 : 16)) == 0;
  if (dt == 0)
    hipLaunchKernelGGL(gla_out_kernel<bf16_t>, grid, dim3(256), 0, st, obuf, (const bf16_t*)gate, gate_stride,
                       (const bf16_t*)w, (bf16_t*)out, out_stride, out_scale, n, NH, V, eps, vec, sigmoid);
  else
    hipLaunchKernelGGL(gla_out_kernel<float>, grid, dim3(256), 0, st, obuf, (const float*)gate, gate_stride,
                       (const float*)w, (float*)out, out_stride, out_scale, n, NH, V, eps, vec, sigmoid);
  return (int)hipGetLastError();
}
