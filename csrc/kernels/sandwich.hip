// Kernels of designs that norm a sublayer's output before it is added (ops/hybrid.py). S = storage
// type (u16 = bf16 bits, or float); the stream, the sublayers' outputs and all arithmetic are
// fp32.
//
//  * sandwich_add    x += rms(y) * (w_post + off);  h = rms(x) * (w_next + off) -> S, in one
//                    launch. y is a row of a GEMM (or the sum of its split-K slabs), the mean of
//                    two rows that are each RMS-normed with a weight of their own (two mixers side
//                    by side), or the sum of a token's routed expert rows and its shared row.
//  * gated_rmsnorm   RMS norm, in equal parts of a row, of y * silu(z), times w -> S
#include "common.h"

namespace {

template <typename S> __device__ __forceinline__ float ldf(const S* p);
template <> __device__ __forceinline__ float ldf<u16>(const u16* p) { return bf2f(*p); }
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }

// V consecutive elements as fp32 (V = 4: 16-byte aligned fp32, 8-byte aligned bf16)
template <int V, typename S> __device__ __forceinline__ void ldv(const S* p, float* v) {
  if constexpr (V == 4 && sizeof(S) == 4) {
    const f32x4 q = *reinterpret_cast<const f32x4*>(p);
    v[0] = q[0]; v[1] = q[1]; v[2] = q[2]; v[3] = q[3];
  } else if constexpr (V == 4) {
    const uint2 b = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(b.x << 16); v[1] = __uint_as_float(b.x & 0xffff0000u);
    v[2] = __uint_as_float(b.y << 16); v[3] = __uint_as_float(b.y & 0xffff0000u);
  } else {
    v[0] = ldf(p);
  }
}
template <int V, typename S> __device__ __forceinline__ void stv(S* p, const float* v) {
  if constexpr (V == 4 && sizeof(S) == 4) {
    *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
  } else if constexpr (V == 4) {
    uint2 pk;
    pk.x = pack2bf(v[0], v[1]);
    pk.y = pack2bf(v[2], v[3]);
    *reinterpret_cast<uint2*>(p) = pk;
  } else if constexpr (sizeof(S) == 2) {
    *p = f2bf(v[0]);
  } else {
    *p = v[0];
  }
}

// block-wide sums of two values at once; `red` holds 32 floats
__device__ __forceinline__ void block_sum2(float& a, float& b, float* red) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
  a = wave_sum(a);
  b = wave_sum(b);
  __syncthreads();
  if (lane == 0) { red[wid] = a; red[16 + wid] = b; }
  __syncthreads();
  a = b = 0.f;
  for (int i = 0; i < nw; ++i) { a += red[i]; b += red[16 + i]; }
}

struct SandwichArgs {
  float* x;
  const void* y; int ldy; int nsplit; long ysplit;   // slabs: nsplit matrices, ysplit apart
  const float* y2; int ldy2;
  const void* w1; const void* w2; float inner_eps;   // pair: weights of y and of y2
  const int* pos; int k;                             // routed: rows of y per token
  const void* w_post; const void* w_next; void* h;
  int dim; float eps, off;
};

enum { PLAIN = 0, PAIR = 1, ROUTED = 2 };

// One workgroup per row; a thread owns columns V (tid + i threads), i < NC, and keeps them in
// registers from the first load to the last store.
template <typename S, typename Y, int V, int NC, int MODE>
__global__ void __launch_bounds__(1024) sandwich_kernel(SandwichArgs a) {
  __shared__ float red[32];
  const long r = blockIdx.x;
  const int nt = blockDim.x, dim = a.dim;
  float v[NC][V], xv[NC][V];
  float s1 = 0.f, s2 = 0.f;
  float u[MODE == PAIR ? NC : 1][V];
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (threadIdx.x + i * nt) * V;
#pragma unroll
    for (int e = 0; e < V; ++e) { v[i][e] = 0.f; xv[i][e] = 0.f; }
    if (MODE == PAIR) {
#pragma unroll
      for (int e = 0; e < V; ++e) u[MODE == PAIR ? i : 0][e] = 0.f;
    }
    if (c >= dim) continue;
    float t[V];
    ldv<V>(a.x + r * dim + c, xv[i]);
    if (MODE == ROUTED) {
      if (a.y2 != nullptr) ldv<V>(a.y2 + r * a.ldy2 + c, v[i]);
      for (int j = 0; j < a.k; ++j) {
        const int p = a.pos[r * a.k + j];
        if (p < 0) continue;
        ldv<V>((const Y*)a.y + (long)p * a.ldy + c, t);
#pragma unroll
        for (int e = 0; e < V; ++e) v[i][e] += t[e];
      }
    } else {
      const float* yp = (const float*)a.y + r * a.ldy + c;
      ldv<V>(yp, v[i]);
#pragma unroll 4
      for (int k = 1; k < a.nsplit; ++k) {
        ldv<V>(yp + k * a.ysplit, t);
#pragma unroll
        for (int e = 0; e < V; ++e) v[i][e] += t[e];
      }
    }
    if constexpr (MODE == PAIR) {
      ldv<V>(a.y2 + r * a.ldy2 + c, u[i]);
#pragma unroll
      for (int e = 0; e < V; ++e) { s1 += v[i][e] * v[i][e]; s2 += u[i][e] * u[i][e]; }
    }
  }
  if constexpr (MODE == PAIR) {
    block_sum2(s1, s2, red);
    const float r1 = 0.5f / sqrtf(s1 / (float)dim + a.inner_eps);
    const float r2 = 0.5f / sqrtf(s2 / (float)dim + a.inner_eps);
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      const int c = (threadIdx.x + i * nt) * V;
      if (c >= dim) continue;
      float wa[V], wb[V];
      ldv<V>((const S*)a.w1 + c, wa);
      ldv<V>((const S*)a.w2 + c, wb);
#pragma unroll
      for (int e = 0; e < V; ++e) v[i][e] = v[i][e] * r1 * wa[e] + u[i][e] * r2 * wb[e];
    }
  }
  float rs = 1.f;
  if (a.w_post != nullptr) {
    s1 = 0.f;
#pragma unroll
    for (int i = 0; i < NC; ++i)
#pragma unroll
      for (int e = 0; e < V; ++e) s1 += v[i][e] * v[i][e];
    rs = 1.f / sqrtf(block_sum(s1, red) / (float)dim + a.eps);
  }
  s1 = 0.f;
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (threadIdx.x + i * nt) * V;
    if (c >= dim) continue;
    float w[V];
    if (a.w_post != nullptr) {
      ldv<V>((const S*)a.w_post + c, w);
#pragma unroll
      for (int e = 0; e < V; ++e) v[i][e] *= rs * (w[e] + a.off);
    }
#pragma unroll
    for (int e = 0; e < V; ++e) {
      xv[i][e] += v[i][e];
      s1 += xv[i][e] * xv[i][e];
    }
    stv<V>(a.x + r * dim + c, xv[i]);
  }
  if (a.h == nullptr) return;
  rs = 1.f / sqrtf(block_sum(s1, red) / (float)dim + a.eps);
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (threadIdx.x + i * nt) * V;
    if (c >= dim) continue;
    float w[V];
    ldv<V>((const S*)a.w_next + c, w);
#pragma unroll
    for (int e = 0; e < V; ++e) xv[i][e] *= rs * (w[e] + a.off);
    stv<V>((S*)a.h + r * dim + c, xv[i]);
  }
}

template <typename S, typename Y, int MODE>
int launch_sandwich(const SandwichArgs& a, int rows, bool v4, hipStream_t st) {
  const int units = v4 ? a.dim / 4 : a.dim;
  // few rows (decode steps) are bound by latency: more threads a row
  int nt = rows <= 1024 ? 1024 : 256;
  while (nt > 64 && nt / 2 >= units) nt /= 2;
  int nc = (units + nt - 1) / nt;
  while (nc > 4 && nt < 1024) { nt *= 2; nc = (units + nt - 1) / nt; }
#define SW_LAUNCH(VV, N) sandwich_kernel<S, Y, VV, N, MODE><<<rows, nt, 0, st>>>(a)
  if (v4) {
    if (nc <= 1) SW_LAUNCH(4, 1);
    else if (nc <= 2) SW_LAUNCH(4, 2);
    else if (nc <= 4) SW_LAUNCH(4, 4);
    else return (int)hipErrorInvalidValue;
  } else {
    if (nc <= 4) SW_LAUNCH(1, 4);
    else if (nc <= 16) SW_LAUNCH(1, 16);
    else return (int)hipErrorInvalidValue;
  }
#undef SW_LAUNCH
  DLI_RETURN_LAUNCH();
}

// One wave per part of a row, NWAVE parts a workgroup; VEC as above. Narrow parts read twice
// (the second read hits the cache).
template <typename S, int V>
__global__ void __launch_bounds__(256) gated_rmsnorm_kernel(
    S* __restrict__ out, const float* __restrict__ src, int lds, const float* __restrict__ gate,
    int ldg, const S* __restrict__ w, long parts, int n, int groups, float eps) {
  const int lane = threadIdx.x & 63;
  const long p = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (p >= parts) return;
  const long t = p / groups;
  const int o = (int)(p % groups) * n;
  const float* sp = src + t * lds + o;
  const float* gp = gate + t * ldg + o;
  constexpr int KEEP = 8;                        // columns kept in registers: 64 V KEEP
  float kept[KEEP][V];
  float ss = 0.f;
  const auto gated = [&](int c, float* v) {
    float g[V];
    ldv<V>(sp + c, v);
    ldv<V>(gp + c, g);
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] *= g[e] / (1.f + expf(-g[e]));
  };
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = (lane + 64 * i) * V;
    if (c >= n) continue;
    gated(c, kept[i]);
#pragma unroll
    for (int e = 0; e < V; ++e) ss += kept[i][e] * kept[i][e];
  }
  for (int c = (lane + 64 * KEEP) * V; c < n; c += 64 * V) {
    float v[V];
    gated(c, v);
#pragma unroll
    for (int e = 0; e < V; ++e) ss += v[e] * v[e];
  }
  const float rs = 1.f / sqrtf(wave_sum(ss) / (float)n + eps);
  S* op = out + t * (long)groups * n + o;
  const auto store = [&](int c, float* v) {
    float ww[V];
    ldv<V>(w + o + c, ww);
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] *= rs * ww[e];
    stv<V>(op + c, v);
  };
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = (lane + 64 * i) * V;
    if (c < n) store(c, kept[i]);
  }
  for (int c = (lane + 64 * KEEP) * V; c < n; c += 64 * V) {
    float v[V];
    gated(c, v);
    store(c, v);
  }
}

// The same with one workgroup per part: few, wide parts (a decode step)
template <typename S>
__global__ void __launch_bounds__(1024) gated_rmsnorm_block_kernel(
    S* __restrict__ out, const float* __restrict__ src, int lds, const float* __restrict__ gate,
    int ldg, const S* __restrict__ w, int n, int groups, float eps) {
  __shared__ float red[16];
  const long t = blockIdx.x / groups;
  const int o = (int)(blockIdx.x % groups) * n;
  float kept[4], ss = 0.f;
  const auto gated = [&](int c) {
    const float g = gate[t * ldg + o + c];
    return src[t * lds + o + c] * (g / (1.f + expf(-g)));
  };
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    kept[i] = c < n ? gated(c) : 0.f;
    ss += kept[i] * kept[i];
  }
  for (int c = threadIdx.x + 4 * blockDim.x; c < n; c += blockDim.x) {
    const float v = gated(c);
    ss += v * v;
  }
  const float rs = 1.f / sqrtf(block_sum(ss, red) / (float)n + eps);
  S* op = out + t * (long)groups * n + o;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = threadIdx.x + i * blockDim.x;
    if (c < n) {
      const float v = kept[i] * rs * ldf(w + o + c);
      stv<1>(op + c, &v);
    }
  }
  for (int c = threadIdx.x + 4 * blockDim.x; c < n; c += blockDim.x) {
    const float v = gated(c) * rs * ldf(w + o + c);
    stv<1>(op + c, &v);
  }
}

}  // namespace

// y: fp32, or with pos (routed rows, k a token) also bf16 (y_bf16). w1 and w2 given: the mean of
// the normed rows of y (weight w1) and y2 (weight w2). w_post null: x += y. w_next null: no h.
extern "C" int dli_sandwich_add(float* x, const void* y, int ldy, int nsplit, long ysplit,
                                const float* y2, int ldy2, const void* w1, const void* w2,
                                float inner_eps, const int* pos, int k, int y_bf16,
                                const void* w_post, const void* w_next, void* h, int rows, int dim,
                                float eps, float off, int dt, hipStream_t st) {
  if (rows <= 0) return 0;
  const bool pair = w1 != nullptr;
  if (x == nullptr || y == nullptr || dim < 1 || dim > 16384 || nsplit < 1 ||
      (w1 == nullptr) != (w2 == nullptr) || (pair && (y2 == nullptr || pos != nullptr)) ||
      (pos != nullptr && (k < 1 || nsplit != 1)) || (pos == nullptr && (y_bf16 || (!pair && y2))) ||
      (w_next == nullptr) != (h == nullptr) || (dt != 0 && dt != 1))
    return (int)hipErrorInvalidValue;
  const uintptr_t mis = (uintptr_t)x | (uintptr_t)y | (uintptr_t)y2 | (uintptr_t)h;
  const uintptr_t misw = (uintptr_t)w1 | (uintptr_t)w2 | (uintptr_t)w_post | (uintptr_t)w_next;
  const bool v4 = dim % 4 == 0 && ldy % 4 == 0 && ysplit % 4 == 0 && (y2 == nullptr || ldy2 % 4 == 0) &&
                  mis % 16 == 0 && misw % 16 == 0;
  SandwichArgs a{x, y, ldy, nsplit, ysplit, y2, ldy2, w1, w2, inner_eps, pos, k, w_post, w_next, h,
                 dim, eps, off};
#define SW_MODE(S)                                                                      \
  if (pair) return launch_sandwich<S, float, PAIR>(a, rows, v4, st);                    \
  if (pos != nullptr)                                                                   \
    return y_bf16 ? launch_sandwich<S, u16, ROUTED>(a, rows, v4, st)                    \
                  : launch_sandwich<S, float, ROUTED>(a, rows, v4, st);                 \
  return launch_sandwich<S, float, PLAIN>(a, rows, v4, st)
  if (dt == 0) { SW_MODE(u16); }
  SW_MODE(float);
#undef SW_MODE
}

extern "C" int dli_gated_rmsnorm(void* out, const float* src, int lds, const float* gate, int ldg,
                                 const void* w, int T, int n, int groups, float eps, int dt,
                                 hipStream_t st) {
  if (T <= 0) return 0;
  if (n < 1 || groups < 1 || out == nullptr || w == nullptr || (dt != 0 && dt != 1))
    return (int)hipErrorInvalidValue;
  const long parts = (long)T * groups;
  if (parts < 1024 && n >= 512) {
    const int nt = n >= 2048 ? 1024 : 256;
    if (dt == 0)
      gated_rmsnorm_block_kernel<u16><<<(int)parts, nt, 0, st>>>((u16*)out, src, lds, gate, ldg,
                                                                 (const u16*)w, n, groups, eps);
    else
      gated_rmsnorm_block_kernel<float><<<(int)parts, nt, 0, st>>>((float*)out, src, lds, gate, ldg,
                                                                   (const float*)w, n, groups, eps);
    DLI_RETURN_LAUNCH();
  }
  const bool v4 = n % 4 == 0 && lds % 4 == 0 && ldg % 4 == 0 &&
                  ((uintptr_t)out | (uintptr_t)src | (uintptr_t)gate | (uintptr_t)w) % 16 == 0;
  const int nb = (int)((parts + 3) / 4);
#define GR_LAUNCH(S, V)                                                                      \
  gated_rmsnorm_kernel<S, V><<<nb, 256, 0, st>>>((S*)out, src, lds, gate, ldg, (const S*)w, parts, \
                                                 n, groups, eps)
  if (v4) { if (dt == 0) GR_LAUNCH(u16, 4); else GR_LAUNCH(float, 4); }
  else { if (dt == 0) GR_LAUNCH(u16, 1); else GR_LAUNCH(float, 1); }
#undef GR_LAUNCH
  DLI_RETURN_LAUNCH();
}
