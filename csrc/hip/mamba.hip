// Selective scan: a diagonal recurrence per channel and state index whose step size, input and read-out weights depend on
// the token.
//
//   dt_t[c]   = softplus(r_t[c] + bias[c])                              r: fp32 rows (a low-rank projection of the token)
//   S_t[n, c] = exp(dt_t[c] A[c, n]) S_(t-1)[n, c] + dt_t[c] x_t[c] B_t[n],     A = -exp(A_log)
//   y_t[c]    = sum_n S_t[n, c] C_t[n] + D[c] x_t[c];   out = y silu(z)
//
// x, z, B, C are rows in the storage type T; step sizes, decays, state and read-out are fp32. State slots [slots, N, I]
// live in device memory between steps: a row whose first token has position 0 starts from S = 0 whatever its slot held
// before; a row with a negative slot is skipped (its outputs are zero).
//
// One workgroup of four waves per (row, 64 channels): lane = channel, wave r keeps a quarter of the state indices in
// registers. The operands of TC tokens are staged in LDS ahead (the next TC are fetched into registers meanwhile), the
// waves' partial read-outs meet in LDS once per TC tokens.
#include "common.hpp"

namespace {

template <typename T> DEVINL float ldf(const T* p, size_t i);
template <> DEVINL float ldf<bf16_t>(const bf16_t* p, size_t i) { return bf2f(p[i]); }
template <> DEVINL float ldf<float>(const float* p, size_t i) { return p[i]; }
template <typename T> DEVINL void stf(T* p, size_t i, float v);
template <> DEVINL void stf<bf16_t>(bf16_t* p, size_t i, float v) { p[i] = f2bf(v); }
template <> DEVINL void stf<float>(float* p, size_t i, float v) { p[i] = v; }

// bf16 storage: hardware exponential and logarithm (a short series where 1 + e would lose e's digits)
template <typename T> DEVINL float softplus(float z) {
  if (sizeof(T) == 2) {
    const float e = __expf(-fabsf(z));
    return fmaxf(z, 0.f) + (e < 0.0156f ? e * (1.f - e * (0.5f - 0.33333333f * e)) : __logf(1.f + e));
  }
  return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));
}
template <typename T> DEVINL float silu(float z) {
  return sizeof(T) == 2 ? z * __builtin_amdgcn_rcpf(1.f + __expf(-z)) : z / (1.f + expf(-z));
}
// bf16 storage: v_exp_f32 (relative error ~1e-6, far below the storage's); fp32 storage: the library's
template <typename T> DEVINL float exp2_le0(float x) { return sizeof(T) == 2 ? fast_exp2(x) : exp2f(x); }
constexpr float LOG2E = 1.4426950408889634f;
constexpr int RW = 4;  // waves of a workgroup

// NP: state indices per wave (a multiple of 2; N <= RW * NP), TC: tokens staged per step
template <typename T, int NP, int TC>
__global__ void __launch_bounds__(64 * RW) selective_scan_kernel(
    const T* __restrict__ x, int64_t x_stride, const float* __restrict__ r, int64_t r_stride, const T* __restrict__ dt_bias,
    const T* __restrict__ a_log, const T* __restrict__ bc, int64_t bc_stride, const T* __restrict__ dskip,
    const T* __restrict__ z, int64_t z_stride, const int* __restrict__ cu_q, const int* __restrict__ first_pos,
    const int* __restrict__ state_slots, float* __restrict__ S, T* __restrict__ out, int I, int N) {
  constexpr int NT = RW * NP;
  constexpr int EC = (TC * 64) / (64 * RW), EN = (TC * NT + 64 * RW - 1) / (64 * RW);
  __shared__ float sdt[TC][64], sdx[TC][64];
  __shared__ __attribute__((aligned(16))) float sB[TC][NT], sC[TC][NT];
  __shared__ float part[RW][TC][64];
  const int b = blockIdx.x, tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int c = blockIdx.y * 64 + lane, cc = min(c, I - 1);
  const bool has = c < I;
  const int slot = state_slots[b], t_lo = cu_q[b], t_hi = cu_q[b + 1];
  if (slot < 0) {
    for (int t = t_lo + w; t < t_hi; t += RW)
      if (has) stf<T>(out, (size_t)t * I + c, 0.f);
    return;
  }
  if (t_hi <= t_lo) return;
  const bool fresh = first_pos[b] == 0;
  float s[NP], a[NP];
#pragma unroll
  for (int k = 0; k < NP; ++k) {
    const int n = w * NP + k;
    const bool live = n < N;
    a[k] = live ? -expf(ldf<T>(a_log, (size_t)cc * N + min(n, N - 1))) * LOG2E : 0.f;
    s[k] = (live && has && !fresh) ? S[((size_t)slot * N + n) * I + c] : 0.f;
  }
  const float bias = ldf<T>(dt_bias, cc), dsk = ldf<T>(dskip, cc);
  // this thread's share of the operands of TC tokens: tokens w, w + RW, ... of its channel; B and C spread over all threads
  float fr[EC], fx[EC], fz[EC], fB[EN], fC[EN];
  auto fetch = [&](int tb) {
#pragma unroll
    for (int e = 0; e < EC; ++e) {
      const size_t t = (size_t)min(tb + w + RW * e, t_hi - 1);
      fr[e] = r[t * r_stride + cc];
      fx[e] = ldf<T>(x, t * x_stride + cc);
      fz[e] = ldf<T>(z, t * z_stride + cc);
    }
#pragma unroll
    for (int e = 0; e < EN; ++e) {
      const int i = tid + 64 * RW * e, n = i % NT, tt = min(i / NT, TC - 1);
      const size_t at = (size_t)min(tb + tt, t_hi - 1) * bc_stride;
      fB[e] = n < N ? ldf<T>(bc, at + n) : 0.f;
      fC[e] = n < N ? ldf<T>(bc, at + N + n) : 0.f;
    }
  };
  fetch(t_lo);
  for (int tb = t_lo; tb < t_hi; tb += TC) {
    const int nt = min(TC, t_hi - tb);
    float cx[EC], cz[EC];
#pragma unroll
    for (int e = 0; e < EC; ++e) {
      // tokens past the row's end leave the state as it is: step size zero
      const float d = tb + w + RW * e < t_hi ? softplus<T>(fr[e] + bias) : 0.f;
      sdt[w + RW * e][lane] = d;
      sdx[w + RW * e][lane] = d * fx[e];
      cx[e] = fx[e];
      cz[e] = fz[e];
    }
#pragma unroll
    for (int e = 0; e < EN; ++e) {
      const int i = tid + 64 * RW * e;
      if (TC * NT % (64 * RW) == 0 || i < TC * NT) {
        sB[i / NT][i % NT] = fB[e];
        sC[i / NT][i % NT] = fC[e];
      }
    }
    if (tb + TC < t_hi) fetch(tb + TC);
    __syncthreads();
#pragma unroll
    for (int tt = 0; tt < TC; ++tt) {
      const float d = sdt[tt][lane], u = sdx[tt][lane];
      float y = 0.f;
#pragma unroll
      for (int k = 0; k < NP; ++k) {
        s[k] = exp2_le0<T>(d * a[k]) * s[k] + u * sB[tt][w * NP + k];
        y += s[k] * sC[tt][w * NP + k];
      }
      part[w][tt][lane] = y;
    }
    __syncthreads();
#pragma unroll
    for (int e = 0; e < EC; ++e) {
      const int tt = w + RW * e;
      if (tt < nt && has) {
        float y = 0.f;
#pragma unroll
        for (int k = 0; k < RW; ++k) y += part[k][tt][lane];
        y += dsk * cx[e];
        stf<T>(out, (size_t)(tb + tt) * I + c, y * silu<T>(cz[e]));
      }
    }
    __syncthreads();  // the partials and the staged operands are free
  }
  if (has) {
#pragma unroll
    for (int k = 0; k < NP; ++k)
      if (w * NP + k < N) S[((size_t)slot * N + w * NP + k) * I + c] = s[k];
  }
}

}  // namespace

// x [T, I] (x_stride), r fp32 [T, I] (r_stride), dt_bias / dskip [I], a_log [I, N], bc rows: N read-in weights, then N
// read-out weights (bc_stride), z [T, I] (z_stride); S [slots, N, I] fp32; out [T, I] contiguous. N <= 256.
extern "C" int areal_selective_scan(const void* x, int64_t x_stride, const float* r, int64_t r_stride,
                                    const void* dt_bias, const void* a_log, const void* bc, int64_t bc_stride,
                                    const void* dskip, const void* z, int64_t z_stride, const int* cu_q,
                                    const int* first_pos, const int* state_slots, float* S, void* out, int B, int I, int N,
                                    int max_q, int dt, hipStream_t st) {
  if (B == 0) return 0;
  if (I <= 0 || N <= 0 || N > 256) return -1;
  const dim3 grid(B, (I + 63) / 64);
#define LAUNCH(TT, NPV, TCV)                                                                                         \
  hipLaunchKernelGGL((selective_scan_kernel<TT, NPV, TCV>), grid, dim3(64 * RW), 0, st, (const TT*)x, x_stride, r,    \
                     r_stride, (const TT*)dt_bias, (const TT*)a_log, (const TT*)bc, bc_stride, (const TT*)dskip,      \
                     (const TT*)z, z_stride, cu_q, first_pos, state_slots, S, (TT*)out, I, N)
#define PICK(TT, TCV)                    \
  do {                                   \
    if (N <= 16) LAUNCH(TT, 4, TCV);     \
    else if (N <= 24) LAUNCH(TT, 6, TCV); \
    else if (N <= 32) LAUNCH(TT, 8, TCV); \
    else if (N <= 64) LAUNCH(TT, 16, TCV); \
    else if (N <= 128) LAUNCH(TT, 32, TCV); \
    else LAUNCH(TT, 64, 4);              \
  } while (0)
#define PICK_TC(TT)             \
  do {                          \
    if (max_q > 4) PICK(TT, 16); \
    else PICK(TT, 4);           \
  } while (0)
  if (dt == 0) PICK_TC(bf16_t);
  else PICK_TC(float);
#undef PICK_TC
#undef PICK
#undef LAUNCH
  return (int)hipGetLastError();
}
