// Element-wise norm ("dynamic tanh") on an fp32 residual stream, and what stands around it:
//
//   N(z) = tanh(alpha * z) * w + b               alpha one number, w and b vectors over the channels; no statistics
//
//   embed_sinusoid   x = E[token] + P(position),  P[2i] = sin(p base^(-2i/W)), P[2i+1] = cos of the same
//   tanh_norm_step   closes a sublayer:   x <- x + N_b(y)
//                    or enters a pass:    x <- p + c + s          (p, c fp32 products, s a vector over the channels)
//                    and hands on either N_next(x) or x itself in the storage type (and N_next(x) in fp32)
//
// y is a tensor in the storage type T, or the sum of fp32 slabs (a split product's partial sums), or the recombination of
// routed experts: y = sum_j wt[t, j] ys[inv[t k + j]] + sigmoid(sg_t) y_sh. Everything is element by element: a thread
// keeps its channels' weights in registers and walks down rows. The angle of a position vector is formed and brought into
// one turn in fp64, its sine and cosine are taken in fp32.
#include "common.hpp"

namespace {

template <typename T, int VEC> DEVINL void ldv(const T* p, size_t i, float (&o)[VEC]) {
  typedef T tv __attribute__((ext_vector_type(VEC)));
  if constexpr (VEC == 1) {
    o[0] = (float)p[i];
  } else {
    const tv x = *reinterpret_cast<const tv*>(p + i);
#pragma unroll
    for (int e = 0; e < VEC; ++e) o[e] = (float)x[e];
  }
}
template <typename T, int VEC> DEVINL void stv(T* p, size_t i, const float (&o)[VEC]) {
  typedef T tv __attribute__((ext_vector_type(VEC)));
  if constexpr (VEC == 1) {
    p[i] = (T)o[0];
  } else {
    tv x;
#pragma unroll
    for (int e = 0; e < VEC; ++e) x[e] = (T)o[e];
    *reinterpret_cast<tv*>(p + i) = x;
  }
}
// weights may sit anywhere in a flat parameter buffer: element loads
template <typename T, int VEC> DEVINL void ldw(const T* p, int i, float (&o)[VEC]) {
#pragma unroll
  for (int e = 0; e < VEC; ++e) o[e] = p ? (float)p[i + e] : 0.f;
}

struct StepArgs {
  const float* x;   // null: a pass is entered (x = p + c + s)
  const void* y;    // T [n, W], or fp32 [slabs, n, W], or (inv set) expert rows T [n k, W]; null: nothing is added
  int slabs;
  const int64_t* inv;
  const float* wt;
  int k;
  const void* y_sh;       // T [n, W] or null
  const float* sg;        // logits, sg_stride apart
  int64_t sg_stride;
  const void *b_alpha, *b_w, *b_b;
  const float *p, *c;
  const void* s;
  const void *n_alpha, *n_w, *n_b;  // null n_w: x itself is handed on in oc (when oc is set)
  float *x_out, *o32;
  void* oc;
  int n, W, rows;  // rows: rows a workgroup walks
};

template <typename T, int VEC>
__global__ void __launch_bounds__(256) tanh_norm_step_kernel(const StepArgs a) {
  const int W = a.W, i = (blockIdx.x * 256 + threadIdx.x) * VEC;
  if (i >= W) return;
  const int t0 = blockIdx.y * a.rows, t1 = min(a.n, t0 + a.rows);
  float bw[VEC], bb[VEC], nw[VEC], nb[VEC];
  const float ba = a.b_alpha ? (float)*(const T*)a.b_alpha : 0.f, na = a.n_alpha ? (float)*(const T*)a.n_alpha : 0.f;
  ldw<T, VEC>((const T*)(a.x ? a.b_w : a.s), i, bw);
  ldw<T, VEC>((const T*)a.b_b, i, bb);
  ldw<T, VEC>((const T*)a.n_w, i, nw);
  ldw<T, VEC>((const T*)a.n_b, i, nb);
  for (int t = t0; t < t1; ++t) {
    const size_t at = (size_t)t * W + i;
    float x[VEC];
    if (a.x) {
      ldv<float, VEC>(a.x, at, x);
      if (a.y) {
        float z[VEC];
        if (a.inv) {
#pragma unroll
          for (int e = 0; e < VEC; ++e) z[e] = 0.f;
          for (int j = 0; j < a.k; ++j) {
            const float wj = a.wt[(size_t)t * a.k + j];
            float r[VEC];
            ldv<T, VEC>((const T*)a.y, (size_t)a.inv[(size_t)t * a.k + j] * W + i, r);
#pragma unroll
            for (int e = 0; e < VEC; ++e) z[e] += wj * r[e];
          }
          if (a.y_sh) {
            const float g = 1.f / (1.f + expf(-a.sg[(size_t)t * a.sg_stride]));
            float r[VEC];
            ldv<T, VEC>((const T*)a.y_sh, at, r);
#pragma unroll
            for (int e = 0; e < VEC; ++e) z[e] += g * r[e];
          }
        } else if (a.slabs > 0) {
          ldv<float, VEC>((const float*)a.y, at, z);
          for (int s = 1; s < a.slabs; ++s) {
            float r[VEC];
            ldv<float, VEC>((const float*)a.y, (size_t)s * a.n * W + at, r);
#pragma unroll
            for (int e = 0; e < VEC; ++e) z[e] += r[e];
          }
        } else {
          ldv<T, VEC>((const T*)a.y, at, z);
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) x[e] += tanhf(ba * z[e]) * bw[e] + bb[e];
      }
    } else {
      float c[VEC];
      ldv<float, VEC>(a.p, at, x);
      ldv<float, VEC>(a.c, at, c);
#pragma unroll
      for (int e = 0; e < VEC; ++e) x[e] = x[e] + c[e] + bw[e];
    }
    if (a.x_out) stv<float, VEC>(a.x_out, at, x);
    if (a.n_w) {
#pragma unroll
      for (int e = 0; e < VEC; ++e) x[e] = tanhf(na * x[e]) * nw[e] + nb[e];
      if (a.o32) stv<float, VEC>(a.o32, at, x);
    }
    if (a.oc) stv<T, VEC>((T*)a.oc, at, x);
  }
}

template <typename T>
__global__ void __launch_bounds__(256) embed_sinusoid_kernel(const int64_t* __restrict__ tokens,
                                                             const int* __restrict__ positions,
                                                             const T* __restrict__ embed, const double* __restrict__ freq,
                                                             int vocab, float* __restrict__ x, T* __restrict__ oc, int W) {
  const size_t t = blockIdx.x;
  int64_t tok = tokens[t];
  tok = tok < 0 ? 0 : (tok >= vocab ? vocab - 1 : tok);
  const double p = (double)max(positions[t], 0);
  for (int i = blockIdx.y * 256 + threadIdx.x; 2 * i < W; i += 256 * gridDim.y) {
    double turn = p * freq[i] * 0.15915494309189533576888;  // 1 / (2 pi)
    turn -= rint(turn);
    float sn, cs;
    sincosf((float)(turn * 6.28318530717958647692529), &sn, &cs);
    const size_t at = t * W + 2 * i;
    const float u = (float)embed[(size_t)tok * W + 2 * i] + sn;
    x[at] = u;
    if (oc) oc[at] = (T)u;
    if (2 * i + 1 < W) {
      const float v = (float)embed[(size_t)tok * W + 2 * i + 1] + cs;
      x[at + 1] = v;
      if (oc) oc[at + 1] = (T)v;
    }
  }
}

// z <- cap tanh(z / cap), in place
template <typename T>
__global__ void __launch_bounds__(256) softcap_kernel(T* __restrict__ z, int64_t n, float cap, float inv) {
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256)
    z[i] = (T)(cap * tanhf((float)z[i] * inv));
}

}  // namespace

// See StepArgs. Rows are [n, W] contiguous; dt 0: bf16, 1: fp32 storage.
extern "C" int areal_tanh_norm_step(const float* x, const void* y, int slabs, const int64_t* inv, const float* wt, int k,
                                    const void* y_sh, const float* sg, int64_t sg_stride, const void* b_alpha,
                                    const void* b_w, const void* b_b, const float* p, const float* c, const void* s,
                                    const void* n_alpha, const void* n_w, const void* n_b, float* x_out, float* o32,
                                    void* oc, int n, int W, int dt, hipStream_t st) {
  if (n == 0) return 0;
  if (W < 1 || (y && (!x || !b_alpha || !b_w || !b_b)) || (!x && (!p || !c || !s))) return -1;
  if ((inv && (!wt || k < 1)) || (y_sh && (!inv || !sg)) || (n_w && (!n_alpha || !n_b))) return -1;
  const uintptr_t a32 = (uintptr_t)x | (uintptr_t)p | (uintptr_t)c | (uintptr_t)x_out | (uintptr_t)o32 |
                        (slabs > 0 ? (uintptr_t)y : 0);
  const uintptr_t at = (slabs > 0 ? 0 : (uintptr_t)y) | (uintptr_t)y_sh | (uintptr_t)oc;
  const bool vec = W % 4 == 0 && a32 % 16 == 0 && at % (dt == 0 ? 8 : 16) == 0;
  const int cols = (W + (vec ? 1024 : 256) - 1) / (vec ? 1024 : 256);
  int rows = (int)(((int64_t)n * cols + 4095) / 4096);  // about 4096 workgroups where there are enough rows
  if (rows < 1) rows = 1;
  if (rows > 16) rows = 16;
  if ((n + rows - 1) / rows > 65535) rows = (n + 65534) / 65535;
  const StepArgs a{x, y, slabs, inv, wt, k, y_sh, sg, sg_stride, b_alpha, b_w, b_b, p, c, s, n_alpha, n_w, n_b,
                   x_out, o32, oc, n, W, rows};
  const dim3 grid(cols, (n + rows - 1) / rows);
#define GO(TT)                                                                                   \
  do {                                                                                           \
    if (vec) hipLaunchKernelGGL((tanh_norm_step_kernel<TT, 4>), grid, dim3(256), 0, st, a);      \
    else hipLaunchKernelGGL((tanh_norm_step_kernel<TT, 1>), grid, dim3(256), 0, st, a);          \
  } while (0)
  if (dt == 0) GO(bf16_t);
  else GO(float);
#undef GO
  return (int)hipGetLastError();
}

// freq fp64 [(W + 1) / 2]; x fp32 [n, W]; oc (or null) the same in the storage type
extern "C" int areal_embed_sinusoid(const int64_t* tokens, const int* positions, const void* embed, const double* freq,
                                    int vocab, float* x, void* oc, int n, int W, int dt, hipStream_t st) {
  if (n == 0) return 0;
  if (W < 1 || vocab < 1) return -1;
  const dim3 grid(n, (W + 2047) / 2048);
  if (dt == 0)
    hipLaunchKernelGGL(embed_sinusoid_kernel<bf16_t>, grid, dim3(256), 0, st, tokens, positions, (const bf16_t*)embed, freq,
                       vocab, x, (bf16_t*)oc, W);
  else
    hipLaunchKernelGGL(embed_sinusoid_kernel<float>, grid, dim3(256), 0, st, tokens, positions, (const float*)embed, freq,
                       vocab, x, (float*)oc, W);
  return (int)hipGetLastError();
}

extern "C" int areal_softcap(void* z, int64_t n, float cap, int dt, hipStream_t st) {
  if (n == 0) return 0;
  if (!(cap > 0.f)) return -1;
  const int64_t want = (n + 255) / 256;
  const dim3 grid((unsigned)(want < 8192 ? want : 8192));
  if (dt == 0) hipLaunchKernelGGL(softcap_kernel<bf16_t>, grid, dim3(256), 0, st, (bf16_t*)z, n, cap, 1.f / cap);
  else hipLaunchKernelGGL(softcap_kernel<float>, grid, dim3(256), 0, st, (float*)z, n, cap, 1.f / cap);
  return (int)hipGetLastError();
}
