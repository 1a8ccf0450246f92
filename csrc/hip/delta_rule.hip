// Gated delta rule with one decay per head and key channel: a matrix state per head, [D, V], kept transposed as [V][D].
//
//   q_t, k_t   unit vectors (x / sqrt(sum x^2 + unit_eps)), q_t times q_scale; head h reads q/k head h / (H / G)
//   ln g_t     = -exp(A_h) * softplus(z_t + bias)         one factor per head and key channel, <= 0
//   beta_t     = sigmoid(b_t)                             one per head
//   S'         = diag(g_t) S_(t-1);   u_t = beta_t (v_t - S'^T k_t);   S_t = S' + k_t u_t^T;   o_t = S_t^T q_t
//
// q, k, v are columns of one tensor (storage type T, after their short convolutions), b columns of another, z fp32
// logits; everything else is fp32. State slots [slots, H, V, D] live in device memory between steps: a row whose first
// token has position 0 starts from S = 0 whatever its slot held before; a row with a negative slot is skipped (its
// outputs are zero).
//
// `delta_scan_kernel` (decoding, short portions, large D): token by token. Columns of S do not talk to each other, so
// eight lanes own a column (an eighth of its D numbers each, as 16-byte pieces) and a token costs two 8-lane sums, which
// run side by side: o_t = S'^T q_t + u_t (k_t . q_t). A workgroup of four waves owns 32 columns; queries, keys and
// factors of up to 8 tokens are staged ahead, one wave a token.
//
// Prompt portions: chunks of 16 tokens. With b_t = sum_{u <= t} ln g_u (per channel, from the chunk's start):
//
//   L[t, s] = beta_t sum_d k_t[d] k_s[d] exp(b_t[d] - b_s[d])  (s < t),      M = (I + L)^-1 diag(beta)
//   U       = M (V - K~ S_0),    K~_t = k_t exp(b_t)
//   o_t     = (q_t exp(b_t))^T S_0 + sum_{s <= t} A[t, s] u_s,               A[t, s] = sum_d q_t[d] k_s[d] exp(b_t[d] - b_s[d])
//   S_new   = diag(exp(b_L)) S_0 + sum_s (k_s exp(b_L - b_s)) u_s^T
//
// Every exponent is <= 0: nothing overflows whatever the decays are, and nothing is divided. `delta_prep_kernel` forms
// what does not depend on the state for all chunks at once; `delta_chunk_kernel` walks a row's chunks with products on
// the fp32 matrix cores (MFMA 16x16x4) only: a wave owns 16 value columns and keeps its slice of the state in registers,
// which are at once the B operand of the products with S_0 and the accumulator of S_new; V - K~ S_0 and U come out of
// one product in the register order in which the next one takes them. Waves share nothing: no LDS, no barriers.
#include "common.hpp"

namespace {

template <typename T> DEVINL float ldf(const T* p, size_t i) { return (float)p[i]; }

// softplus and exp; bf16 storage: hardware exponential and logarithm (a short series where 1 + e would lose e's digits)
template <typename T> DEVINL float softplus(float x) {
  if (sizeof(T) == 2) {
    const float e = __expf(-fabsf(x));
    return fmaxf(x, 0.f) + (e < 0.0156f ? e * (1.f - e * (0.5f - 0.33333333f * e)) : __logf(1.f + e));
  }
  return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x)));
}
// x <= 0. bf16 storage: v_exp_f32 (relative error ~1e-6, far below the storage's); fp32 storage: the library's exp
template <typename T> DEVINL float exp_le0(float x) { return sizeof(T) == 2 ? __expf(x) : expf(x); }

constexpr int CT = 16;  // tokens of a chunk

struct DeltaArgs {
  const void* qkv;
  int64_t row_stride;
  int q_off, k_off, v_off;
  const float* z;
  int64_t z_stride;
  const void *z_bias, *a_log;  // [H D], [H]
  const void* beta;            // logits, [T, H] rows beta_stride apart
  int64_t beta_stride;
  float q_scale, unit_eps;
  const int *cu_q, *first_pos, *state_slots;
  float *S, *obuf, *scratch;
  int H, G, D, V;
};

// CG: columns a lane works on (32 apart): decoding takes two, so that twice the state is under way per wave.
template <typename T, int DP, int TC, int CG>
__global__ void __launch_bounds__(256) delta_scan_kernel(const DeltaArgs a) {
  constexpr int NV = DP / 32;  // 16-byte pieces of a column a lane owns: channels 32 p + 4 l8 .. + 3
  constexpr int NQ = (DP + 63) / 64;
  __shared__ __attribute__((aligned(16))) float kqg[TC][3][DP];
  __shared__ float bet[TC], kq[TC];
  const int H = a.H, G = a.G, D = a.D, V = a.V;
  const int b = blockIdx.x, hd = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int l8 = lane & 7, col = blockIdx.z * 32 * CG + 8 * wave + (lane >> 3), hk = hd / (H / G);
  const int slot = a.state_slots[b], t_lo = a.cu_q[b], t_hi = a.cu_q[b + 1];
  if (slot < 0) {
#pragma unroll
    for (int c = 0; c < CG; ++c)
      if (col + 32 * c < V && l8 == 0)
        for (int t = t_lo; t < t_hi; ++t) a.obuf[((size_t)t * H + hd) * V + col + 32 * c] = 0.f;
    return;
  }
  if (t_hi <= t_lo) return;
  const T* qkv = (const T*)a.qkv;
  const bool fresh = a.first_pos[b] == 0, vec = D % 4 == 0;
  const float decay_rate = -expf(ldf<T>((const T*)a.a_log, hd));
  float vv[CG][TC];
  struct Token {  // what one lane loads of one token
    float q[NQ], k[NQ], z[NQ], b;
  };
  auto load = [&](Token& o, int t) {
    const T* row = qkv + (size_t)t * a.row_stride;
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
      const int d = lane + 64 * i;
      o.q[i] = d < D ? ldf<T>(row, a.q_off + hk * D + d) : 0.f;
      o.k[i] = d < D ? ldf<T>(row, a.k_off + hk * D + d) : 0.f;
      o.z[i] = d < D ? a.z[(size_t)t * a.z_stride + hd * D + d] + ldf<T>((const T*)a.z_bias, hd * D + d) : 0.f;
    }
    o.b = ldf<T>((const T*)a.beta, (size_t)t * a.beta_stride + hd);
  };
  auto stage = [&](const Token& o, int tt) {
    float qq = 0.f, kk = 0.f, qk = 0.f;
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
      qq += o.q[i] * o.q[i];
      kk += o.k[i] * o.k[i];
      qk += o.q[i] * o.k[i];
    }
    const float rq = a.q_scale / sqrtf(wave_sum(qq) + a.unit_eps), rk = 1.f / sqrtf(wave_sum(kk) + a.unit_eps);
    const float dot = wave_sum(qk) * rq * rk;
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
      const int d = lane + 64 * i;
      if (d < DP) {
        kqg[tt][0][d] = o.k[i] * rk;
        kqg[tt][1][d] = o.q[i] * rq;
        kqg[tt][2][d] = d < D ? exp_le0<T>(decay_rate * softplus<T>(o.z[i])) : 0.f;
      }
    }
    if (lane == 0) {
      bet[tt] = 1.f / (1.f + expf(-o.b));
      kq[tt] = dot;
    }
  };
  auto load_v = [&](int tb, int nt) {
#pragma unroll
    for (int tt = 0; tt < TC; ++tt)
#pragma unroll
      for (int c = 0; c < CG; ++c)
        vv[c][tt] = (tt < nt && col + 32 * c < V)
                        ? ldf<T>(qkv + (size_t)(tb + tt) * a.row_stride, a.v_off + hd * V + col + 32 * c) : 0.f;
  };
  // the first tokens' operands are asked for ahead of the state: loads return in order, and the operands' sums and
  // exponentials run while the state arrives
  Token first;
  int nt = min(TC, t_hi - t_lo);
  if (wave < nt) load(first, t_lo + wave);
  load_v(t_lo, nt);
  float* const Sh = a.S + ((size_t)slot * H + hd) * V * D;
  f32x4 s[CG][NV];
#pragma unroll
  for (int c = 0; c < CG; ++c) {
    const float* Sp = Sh + (size_t)min(col + 32 * c, V - 1) * D;
#pragma unroll
    for (int p = 0; p < NV; ++p) {
      const int d = 32 * p + 4 * l8;
      s[c][p] = (f32x4){0.f, 0.f, 0.f, 0.f};
      if (!fresh && col + 32 * c < V) {
        if (vec) {
          if (d < D) s[c][p] = *reinterpret_cast<const f32x4*>(Sp + d);
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (d + e < D) s[c][p][e] = Sp[d + e];
        }
      }
    }
  }
  if (wave < nt) stage(first, wave);
  for (int tb = t_lo; tb < t_hi; tb += TC) {
    nt = min(TC, t_hi - tb);
    if (tb > t_lo) {
      __syncthreads();  // the tokens before are consumed
      load_v(tb, nt);
    }
    for (int tt = wave + (tb == t_lo ? 4 : 0); tt < nt; tt += 4) {
      Token o;
      load(o, tb + tt);
      stage(o, tt);
    }
    __syncthreads();
#pragma unroll
    for (int tt = 0; tt < TC; ++tt) {
      if (tt < nt) {
        f32x4 k4[NV];
        float sk[CG], sq[CG];
#pragma unroll
        for (int c = 0; c < CG; ++c) sk[c] = sq[c] = 0.f;
#pragma unroll
        for (int p = 0; p < NV; ++p) {
          const int d = 32 * p + 4 * l8;
          k4[p] = *reinterpret_cast<const f32x4*>(&kqg[tt][0][d]);
          const f32x4 q4 = *reinterpret_cast<const f32x4*>(&kqg[tt][1][d]), g4 = *reinterpret_cast<const f32x4*>(&kqg[tt][2][d]);
#pragma unroll
          for (int c = 0; c < CG; ++c)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              s[c][p][e] *= g4[e];
              sk[c] += s[c][p][e] * k4[p][e];
              sq[c] += s[c][p][e] * q4[e];
            }
        }
#pragma unroll
        for (int o = 4; o > 0; o >>= 1)
#pragma unroll
          for (int c = 0; c < CG; ++c) {
            sk[c] += __shfl_xor(sk[c], o, 64);
            sq[c] += __shfl_xor(sq[c], o, 64);
          }
#pragma unroll
        for (int c = 0; c < CG; ++c) {
          const float u = bet[tt] * (vv[c][tt] - sk[c]);
#pragma unroll
          for (int p = 0; p < NV; ++p)
#pragma unroll
            for (int e = 0; e < 4; ++e) s[c][p][e] += k4[p][e] * u;
          if (col + 32 * c < V && l8 == 0) a.obuf[((size_t)(tb + tt) * H + hd) * V + col + 32 * c] = sq[c] + u * kq[tt];
        }
      }
    }
  }
#pragma unroll
  for (int c = 0; c < CG; ++c) {
    if (col + 32 * c >= V) continue;
    float* Sp = Sh + (size_t)(col + 32 * c) * D;
#pragma unroll
    for (int p = 0; p < NV; ++p) {
      const int d = 32 * p + 4 * l8;
      if (vec) {
        if (d < D) *reinterpret_cast<f32x4*>(Sp + d) = s[c][p];
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (d + e < D) Sp[d + e] = s[c][p][e];
      }
    }
  }
}

// Slot of the chunk that starts at token tb of row b (first token t_lo) in the scratch buffer; T / CT + B + 1 slots. Per
// (slot, head): q~ [CT][DP], k~ [CT][DP], (k exp(b_L - b))^T [DP][CT], exp(b_L) [DP], A [CT][CT], M [CT][CT].
DEVINL size_t chunk_slot(int t_lo, int tb, int b) { return (size_t)(t_lo / CT + b + (tb - t_lo) / CT); }
template <int DP> constexpr size_t chunk_floats() { return 3 * CT * DP + DP + 2 * CT * CT; }

template <typename T, int DP>
__global__ void __launch_bounds__(256) delta_prep_kernel(const DeltaArgs a) {
  constexpr int QS = DP + 1;  // odd stride: the pair loop's 16 key rows fall on different banks
  __shared__ float Qr[CT * QS], Kr[CT * QS], Bs[CT * QS], rq[CT], rk[CT], bet[CT], Ls[CT][CT + 1];
  const int H = a.H, D = a.D;
  const int b = blockIdx.y, hd = blockIdx.z, tid = threadIdx.x, hk = hd / (H / a.G);
  const int t_lo = a.cu_q[b], t_hi = a.cu_q[b + 1], tb = t_lo + CT * blockIdx.x;
  if (tb >= t_hi || a.state_slots[b] < 0) return;
  const int nt = min(CT, t_hi - tb);
  const T* qkv = (const T*)a.qkv;
  const float decay_rate = -expf(ldf<T>((const T*)a.a_log, hd));
  for (int i = tid; i < CT * DP; i += 256) {
    const int d = i % DP, tt = i / DP;
    const bool live = tt < nt && d < D;
    const size_t tok = (size_t)(tb + min(tt, nt - 1));
    const T* row = qkv + tok * a.row_stride;
    const int dc = min(d, D - 1);
    Kr[tt * QS + d] = live ? ldf<T>(row, a.k_off + hk * D + dc) : 0.f;
    Qr[tt * QS + d] = live ? ldf<T>(row, a.q_off + hk * D + dc) : 0.f;
    // rows past the chunk's end and padding channels do not decay
    Bs[tt * QS + d] =
        live ? decay_rate * softplus<T>(a.z[tok * a.z_stride + hd * D + dc] + ldf<T>((const T*)a.z_bias, hd * D + dc)) : 0.f;
  }
  if (tid < CT) bet[tid] = tid < nt ? 1.f / (1.f + expf(-ldf<T>((const T*)a.beta, (size_t)(tb + tid) * a.beta_stride + hd))) : 0.f;
  __syncthreads();
  {  // lengths of the queries and keys: sixteen neighbouring lanes a token
    const int t = tid / CT, l = tid % CT;
    float qq = 0.f, kk = 0.f;
#pragma unroll
    for (int d = l; d < DP; d += 16) {
      const float x = Qr[t * QS + d], y = Kr[t * QS + d];
      qq += x * x;
      kk += y * y;
    }
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) {
      qq += __shfl_xor(qq, o, 64);
      kk += __shfl_xor(kk, o, 64);
    }
    if (l == 0) {
      rq[t] = a.q_scale / sqrtf(qq + a.unit_eps);
      rk[t] = 1.f / sqrtf(kk + a.unit_eps);
    }
  }
  if (tid < DP) {  // running sums along the chunk's tokens, one channel a thread
    float run = 0.f;
#pragma unroll
    for (int tt = 0; tt < CT; ++tt) {
      run += Bs[tt * QS + tid];
      Bs[tt * QS + tid] = run;
    }
  }
  __syncthreads();
  float* qd = a.scratch + (chunk_slot(t_lo, tb, b) * H + hd) * chunk_floats<DP>();
  float *kt = qd + CT * DP, *kd = kt + CT * DP, *el = kd + CT * DP, *abuf = el + DP, *mbuf = abuf + CT * CT;
  {  // the chunk's own pairs: thread (t, s), s <= t
    const int t = tid / CT, sx = tid % CT;
    float a0 = 0.f, a1 = 0.f;
    if (sx <= t && t < nt) {
      const float *qt = Qr + t * QS, *kk = Kr + t * QS, *ks = Kr + sx * QS, *bt = Bs + t * QS, *bs = Bs + sx * QS;
#pragma unroll 4
      for (int d = 0; d < DP; ++d) {
        const float w = ks[d] * exp_le0<T>(bt[d] - bs[d]);
        a0 += qt[d] * w;
        a1 += kk[d] * w;
      }
      a0 *= rq[t] * rk[sx];
      a1 *= rk[t] * rk[sx];
    }
    abuf[tid] = a0;
    Ls[t][sx] = sx < t ? bet[t] * a1 : 0.f;
  }
  __syncthreads();
  if (tid < CT) {  // column `tid` of (I + L)^-1 diag(beta), by forward substitution
    float x[CT];
#pragma unroll
    for (int t = 0; t < CT; ++t) {
      float r = t == tid ? bet[tid] : 0.f;
#pragma unroll
      for (int s = 0; s < t; ++s) r -= Ls[t][s] * x[s];
      x[t] = r;
      mbuf[t * CT + tid] = r;
    }
  }
  for (int i = tid; i < CT * DP; i += 256) {
    const int d = i % DP, tt = i / DP;
    const float e = exp_le0<T>(Bs[tt * QS + d]);
    qd[i] = Qr[tt * QS + d] * rq[tt] * e;
    kt[i] = Kr[tt * QS + d] * rk[tt] * e;
    const int ks = i % CT, kc = i / CT;
    kd[i] = Kr[ks * QS + kc] * rk[ks] * exp_le0<T>(Bs[(CT - 1) * QS + kc] - Bs[ks * QS + kc]);
  }
  for (int i = tid; i < DP; i += 256) el[i] = exp_le0<T>(Bs[(CT - 1) * QS + i]);
}

template <typename T, int DP>
__global__ void __launch_bounds__(256) delta_chunk_kernel(const DeltaArgs a) {
  constexpr int NB = DP / 16;  // blocks of 16 state rows
  const int H = a.H, D = a.D, V = a.V;
  const int b = blockIdx.x, hd = blockIdx.y, lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int r16 = lane & 15, quad = lane >> 4, c = blockIdx.z * 64 + 16 * w + r16;
  const bool has = c < V;
  const int slot = a.state_slots[b];
  const int t_lo = a.cu_q[b], t_hi = a.cu_q[b + 1];
  if (slot < 0) {
    for (int t = t_lo + quad; t < t_hi; t += 4)
      if (has) a.obuf[((size_t)t * H + hd) * V + c] = 0.f;
    return;
  }
  if (t_hi <= t_lo || blockIdx.z * 64 + 16 * w >= V) return;
  const bool fresh = a.first_pos[b] == 0, vec = D % 4 == 0;
  float* Sp = a.S + (((size_t)slot * H + hd) * V + min(c, V - 1)) * D;
  f32x4 s[NB];
#pragma unroll
  for (int rb = 0; rb < NB; ++rb) {
    const int d = 16 * rb + 4 * quad;
    s[rb] = (f32x4){0.f, 0.f, 0.f, 0.f};
    if (!fresh && has) {
      if (vec) {
        if (d < D) s[rb] = *reinterpret_cast<const f32x4*>(Sp + d);
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (d + i < D) s[rb][i] = Sp[d + i];
      }
    }
  }
  struct Operands {
    f32x4 q[NB], k[NB], kd[NB], e[NB], a, m;
    T v[4];  // as loaded: nothing waits for a load before its chunk's turn
  };
  const T* vp = (const T*)a.qkv + a.v_off + hd * V + min(c, V - 1);
  auto fetch = [&](Operands& o, int tb) {
    const float* base = a.scratch + (chunk_slot(t_lo, tb, b) * H + hd) * chunk_floats<DP>();
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      o.q[i] = *reinterpret_cast<const f32x4*>(base + r16 * DP + 16 * i + 4 * quad);
      o.k[i] = *reinterpret_cast<const f32x4*>(base + CT * DP + r16 * DP + 16 * i + 4 * quad);
      o.kd[i] = *reinterpret_cast<const f32x4*>(base + 2 * CT * DP + (16 * i + r16) * CT + 4 * quad);
      o.e[i] = *reinterpret_cast<const f32x4*>(base + 3 * CT * DP + 16 * i + 4 * quad);
    }
    o.a = *reinterpret_cast<const f32x4*>(base + 3 * CT * DP + DP + r16 * CT + 4 * quad);
    o.m = *reinterpret_cast<const f32x4*>(base + 3 * CT * DP + DP + CT * CT + r16 * CT + 4 * quad);
#pragma unroll
    for (int i = 0; i < 4; ++i)  // rows past the chunk's end meet zeros in M: any finite value will do
      o.v[i] = vp[(size_t)min(tb + 4 * quad + i, t_hi - 1) * a.row_stride];
  };
  auto chunk = [&](const Operands& o, int tb) {
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    f32x4 x0 = zero, x1 = zero, y0 = zero, y1 = zero;
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      x0 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.k[i][0], s[i][0], x0, 0, 0, 0);
      x1 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.k[i][1], s[i][1], x1, 0, 0, 0);
      x0 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.k[i][2], s[i][2], x0, 0, 0, 0);
      x1 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.k[i][3], s[i][3], x1, 0, 0, 0);
    }
    f32x4 x;
#pragma unroll
    for (int i = 0; i < 4; ++i) x[i] = (float)o.v[i] - (x0[i] + x1[i]);
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      y0 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.q[i][0], s[i][0], y0, 0, 0, 0);
      y1 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.q[i][1], s[i][1], y1, 0, 0, 0);
      y0 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.q[i][2], s[i][2], y0, 0, 0, 0);
      y1 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.q[i][3], s[i][3], y1, 0, 0, 0);
    }
    f32x4 u0 = zero, u1 = zero;
    u0 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.m[0], x[0], u0, 0, 0, 0);
    u1 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.m[1], x[1], u1, 0, 0, 0);
    u0 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.m[2], x[2], u0, 0, 0, 0);
    u1 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.m[3], x[3], u1, 0, 0, 0);
    const f32x4 u = u0 + u1;
#pragma unroll
    for (int rb = 0; rb < NB; ++rb) s[rb] *= o.e[rb];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int rb = 0; rb < NB; ++rb) s[rb] = __builtin_amdgcn_mfma_f32_16x16x4f32(o.kd[rb][i], u[i], s[rb], 0, 0, 0);
    y0 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.a[0], u[0], y0, 0, 0, 0);
    y1 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.a[1], u[1], y1, 0, 0, 0);
    y0 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.a[2], u[2], y0, 0, 0, 0);
    y1 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.a[3], u[3], y1, 0, 0, 0);
    y0 += y1;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = tb + 4 * quad + i;
      if (t < t_hi && has) a.obuf[((size_t)t * H + hd) * V + c] = y0[i];
    }
  };
  Operands o0, o1;  // a chunk's loads are under way while the chunk before is worked on
  fetch(o0, t_lo);
  for (int tb = t_lo; tb < t_hi; tb += 2 * CT) {
    if (tb + CT < t_hi) fetch(o1, tb + CT);
    chunk(o0, tb);
    if (tb + CT >= t_hi) break;
    if (tb + 2 * CT < t_hi) fetch(o0, tb + 2 * CT);
    chunk(o1, tb + CT);
  }
#pragma unroll
  for (int rb = 0; rb < NB; ++rb) {
    const int d = 16 * rb + 4 * quad;
    if (!has) continue;
    if (vec) {
      if (d < D) *reinterpret_cast<f32x4*>(Sp + d) = s[rb];
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (d + i < D) Sp[d + i] = s[rb][i];
    }
  }
}

}  // namespace

// Floats of the chunked form's scratch.
extern "C" int64_t areal_delta_scratch(int T, int B, int H, int D) {
  const size_t per = D <= 32 ? chunk_floats<32>() : (D <= 64 ? chunk_floats<64>() : chunk_floats<128>());
  return (int64_t)(T / CT + B + 1) * H * per;
}

// qkv rows hold (at q_off / k_off / v_off) G query heads of D, G key heads of D, H value heads of V. z fp32 rows of H D
// decay logits, z_bias [H D], a_log [H], beta rows of H logits in the storage type `dt` (0: bf16, 1: fp32). S
// [slots, H, V, D] fp32, 16-byte aligned; obuf [T, H, V] fp32. scratch: areal_delta_scratch floats, 16-byte aligned, for
// the chunked form (rows of 16 tokens and more, D <= 128), or null: token by token.
extern "C" int areal_delta_scan(const void* qkv, int64_t row_stride, int q_off, int k_off, int v_off, const float* z,
                                int64_t z_stride, const void* z_bias, const void* a_log, const void* beta,
                                int64_t beta_stride, float q_scale, float unit_eps, const int* cu_q, const int* first_pos,
                                const int* state_slots, float* S, float* obuf, float* scratch, int T, int B, int H, int G,
                                int D, int V, int max_q, int dt, hipStream_t st) {
  if (B == 0 || T == 0) return 0;
  if (D > 256 || D <= 0 || V <= 0 || H <= 0 || G <= 0 || H % G != 0) return -1;
  const DeltaArgs a{qkv, row_stride, q_off, k_off, v_off, z, z_stride, z_bias, a_log, beta, beta_stride, q_scale,
                    unit_eps, cu_q, first_pos, state_slots, S, obuf, scratch, H, G, D, V};
  if (max_q >= CT && D <= 128 && scratch) {
    const dim3 pgrid((max_q + CT - 1) / CT, B, H), grid(B, H, (V + 63) / 64);
#define CHUNK(TT, DPV)                                                              \
  do {                                                                              \
    hipLaunchKernelGGL((delta_prep_kernel<TT, DPV>), pgrid, dim3(256), 0, st, a);   \
    hipLaunchKernelGGL((delta_chunk_kernel<TT, DPV>), grid, dim3(256), 0, st, a);   \
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
  const dim3 grid(B, H, (V + 31) / 32), grid2(B, H, (V + 63) / 64);
#define LAUNCH(TT, DPV)                                                                                   \
  do {                                                                                                    \
    if (max_q == 1) hipLaunchKernelGGL((delta_scan_kernel<TT, DPV, 1, 2>), grid2, dim3(256), 0, st, a);   \
    else hipLaunchKernelGGL((delta_scan_kernel<TT, DPV, 8, 1>), grid, dim3(256), 0, st, a);               \
  } while (0)
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
