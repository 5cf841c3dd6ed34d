// State-space recurrence over per-sequence slots (ops.hybrid.ssd). Per head h (of group g), with a
// step size s_t = softplus(dt_t + dt_bias) and a decay a_t = exp(-rate s_t) per token,
//     S_t = a_t S_{t-1} + s_t B_t x_t^T,      y_t = S_t^T C_t + skip x_t         S [N, P]
// where x [P] is the head's, B and C [N] are the group's, and x, B, C are what a short causal
// filter per channel, a bias and SiLU leave of a projection. A step's tokens of one sequence are
// consecutive rows [cu[s], cu[s+1]) at consecutive positions; state fp32 [slots, H, N, P].
//
// The filter's past is a ring per slot, conv fp32 [slots, taps, channels]: row p mod taps holds the
// input at position p. A token never reads the row it writes, and rows that lie before position 0
// are never read, so neither a reused slot nor the order of workgroups matters.
//
//  * ssd_conv    portions: filter + bias + SiLU of channels x | B | C -> rows [T, channels] (S)
//  * ssd_chunk   portions, in chunks of C tokens. With L_i = sum_{t <= i} log a_t from the chunk's
//                start,
//                  y_i = e^(L_i) S_0^T C_i + sum_{j <= i} e^(L_i - L_j) s_j (B_j . C_i) x_j
//                  S_n = e^(L_n) S_0 + sum_j e^(L_n - L_j) s_j B_j x_j^T
//                four products on the fp32 matrix cores (v_mfma_f32_16x16x4_f32), laid out as in
//                retention.hip: one workgroup of 8 waves per (head, sequence, 64 state columns)
//                walks the chunks, the state stays in the accumulators of the last product and,
//                transposed, in LDS, and the next chunk's rows are in flight in registers. The
//                skip rides on the diagonal of the key-query products. L is summed in double and
//                kept as two floats, so that L_i - L_j loses nothing when decays are strong.
//  * ssd_step    one token a sequence (decode steps), everything in one launch: filter, step size,
//                state (streamed through registers: one read and one write per element), read-out
//
// Sizes the chunk form does not take run the walk of recurrent_scalar.hip.
#include "common.h"

namespace {

constexpr int CW = 64;            // state columns of a workgroup
constexpr int NTH = 512;          // 8 waves
constexpr int PAD = 8;

__device__ __forceinline__ float silu32(float g) { return g / (1.f + expf(-g)); }
__device__ __forceinline__ float softplus32(float z) {
  return z > 0.f ? z + log1pf(expf(-z)) : log1pf(expf(z));
}

// ------------------------------------------------------------------------------ filter
struct ConvArgs {
  const float* u; int ldu;                 // inputs, [T, channels]
  const float* w; const float* b; int taps;
  float* ring;
  const int* slots; const int* cu; const int* positions;
  void* out; int ch, tb;                   // tb: tokens a workgroup filters
};

// Thread = V channels, `tb` tokens in a row through a window in registers (TAPS > 0) or, for
// other tap counts, re-reading the rows. The workgroup of a portion's first tokens also brings
// the ring up to date, after it has read it: same thread, same channels.
template <typename S, int V, int TAPS>
__global__ void __launch_bounds__(256) ssd_conv_kernel(ConvArgs a) {
  const int s = blockIdx.y, t0 = a.cu[s], t1 = a.cu[s + 1];
  const int b0 = t0 + blockIdx.x * a.tb;
  const int c = (blockIdx.z * 256 + threadIdx.x) * V;
  if (b0 >= t1 || c >= a.ch) return;
  const int b1 = min(b0 + a.tb, t1);
  const int slot = a.slots[s], p0 = a.positions[t0];
  const int taps = TAPS ? TAPS : a.taps;
  float* ring = a.ring + (long)max(slot, 0) * taps * a.ch + c;
  const auto load = [&](int t, float* v) {        // the input at row t of the step (or before it)
    const int p = p0 + (t - t0);
    const float* src = t >= t0 ? a.u + (long)t * a.ldu + c
                               : ring + (long)(p >= 0 ? p % taps : 0) * a.ch;
    if (t < t0 && (p < 0 || slot < 0)) {
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] = 0.f;
      return;
    }
    if constexpr (V == 4) {
      const f32x4 q = *reinterpret_cast<const f32x4*>(src);
      v[0] = q[0]; v[1] = q[1]; v[2] = q[2]; v[3] = q[3];
    } else {
      v[0] = *src;
    }
  };
  const auto store = [&](int t, const float* v) {
    S* o = (S*)a.out + (long)t * a.ch + c;
    float y[V];
#pragma unroll
    for (int e = 0; e < V; ++e) y[e] = silu32(v[e]);
    if constexpr (V == 4 && sizeof(S) == 2) {
      uint2 pk;
      pk.x = pack2bf(y[0], y[1]);
      pk.y = pack2bf(y[2], y[3]);
      *reinterpret_cast<uint2*>(o) = pk;
    } else if constexpr (V == 4) {
      *reinterpret_cast<f32x4*>(o) = f32x4{y[0], y[1], y[2], y[3]};
    } else if constexpr (sizeof(S) == 2) {
      *o = f2bf(y[0]);
    } else {
      *o = y[0];
    }
  };
  float bias[V];
#pragma unroll
  for (int e = 0; e < V; ++e) bias[e] = a.b[c + e];
  if constexpr (TAPS > 0) {
    float w[V][TAPS], win[TAPS][V];
#pragma unroll
    for (int e = 0; e < V; ++e)
#pragma unroll
      for (int k = 0; k < TAPS; ++k) w[e][k] = a.w[(long)(c + e) * TAPS + k];
#pragma unroll
    for (int k = 0; k + 1 < TAPS; ++k) load(b0 - TAPS + 1 + k, win[k]);
#pragma unroll 4
    for (int t = b0; t < b1; ++t) {
      load(t, win[TAPS - 1]);
      float acc[V];
#pragma unroll
      for (int e = 0; e < V; ++e) {
        acc[e] = bias[e];
#pragma unroll
        for (int k = 0; k < TAPS; ++k) acc[e] += w[e][k] * win[k][e];
      }
      store(t, acc);
#pragma unroll
      for (int k = 0; k + 1 < TAPS; ++k)
#pragma unroll
        for (int e = 0; e < V; ++e) win[k][e] = win[k + 1][e];
    }
  } else {
    for (int t = b0; t < b1; ++t) {
      float acc[V], v[V];
#pragma unroll
      for (int e = 0; e < V; ++e) acc[e] = bias[e];
      for (int k = 0; k < taps; ++k) {
        load(t - taps + 1 + k, v);
#pragma unroll
        for (int e = 0; e < V; ++e) acc[e] += a.w[(long)(c + e) * taps + k] * v[e];
      }
      store(t, acc);
    }
  }
  if (blockIdx.x != 0 || slot < 0) return;
  for (int t = max(t0, t1 - taps); t < t1; ++t) {
    float v[V];
    load(t, v);
    float* r = ring + (long)((p0 + (t - t0)) % taps) * a.ch;
#pragma unroll
    for (int e = 0; e < V; ++e) r[e] = v[e];
  }
}

// ------------------------------------------------------------------------------ chunks
struct SsdArgs {
  const void* xc; int ldx;                 // filtered rows x [H*P] | B [G*N] | C [G*N]
  const float* dt; int ldt;                // [T, H]
  const float* dt_bias; const float* rate; const float* skip;
  float* state;
  const int* slots; const int* cu; const int* positions;
  float* y;                                // [T, H*P]
  int H, N, P, G;
};

// eight consecutive elements of a filtered row
template <typename S> struct Row8;
template <> struct Row8<float> {
  f32x4 a, b;
  __device__ __forceinline__ void load(const float* p) {
    a = *reinterpret_cast<const f32x4*>(p);
    b = *reinterpret_cast<const f32x4*>(p + 4);
  }
  __device__ __forceinline__ void get(f32x4& x, f32x4& y) const { x = a; y = b; }
};
template <> struct Row8<u16> {
  uint4 v;
  __device__ __forceinline__ void load(const u16* p) { v = *reinterpret_cast<const uint4*>(p); }
  __device__ __forceinline__ void get(f32x4& x, f32x4& y) const {
    float f[8];
    unpack8bf(v, f);
    x = f32x4{f[0], f[1], f[2], f[3]};
    y = f32x4{f[4], f[5], f[6], f[7]};
  }
};
__device__ __forceinline__ f32x4 load4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ f32x4 load4(const u16* p) {
  const uint2 b = *reinterpret_cast<const uint2*>(p);
  return f32x4{__uint_as_float(b.x << 16), __uint_as_float(b.x & 0xffff0000u),
               __uint_as_float(b.y << 16), __uint_as_float(b.y & 0xffff0000u)};
}

// C tokens a chunk; NT: 16-row state tiles a wave accumulates (N <= 32 NT); D: N when it is known
// at compile time (else 0)
template <typename S, int C, int NT, int D>
__global__ void __launch_bounds__(NTH) ssd_chunk_kernel(SsdArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int N = D ? D : a.N, P = a.P, H = a.H, G = a.G;
  const int ldq = N + PAD;
  constexpr int ldc = C + PAD;
  float* Qs = sm;                          // [C][ldq] output vectors C_i
  float* Ks = Qs + C * ldq;                // [C][ldq] input vectors B_j
  float* Vt = Ks + C * ldq;                // [CW][ldc] x, transposed
  float* Ps = Vt + CW * ldc;               // [C][ldc] decayed products (query rows)
  float* St = Ps + C * ldc;                // [CW][ldq] the state before the chunk, transposed
  float* lh = St + CW * ldq;               // [C] L, rounded
  float* ll = lh + C;                      // [C] ... and what rounding left
  float* sz = ll + C;                      // [C] step sizes
  float* eL = sz + C;                      // [C] e^(L_i)
  float* ew = eL + C;                      // [C] e^(L_n - L_j) s_j
  float* en = ew + C;                      // [4] e^(L_n)
  const int h = blockIdx.x, s = blockIdx.y, c0 = blockIdx.z * CW;
  const int ncol = min(CW, P - c0);
  const int slot = a.slots[s], t0 = a.cu[s], t1 = a.cu[s + 1];
  if (t1 <= t0) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int fr = lane & 15, q = lane >> 4;
  const int g = h / (H / G);
  if (slot < 0) {                          // padding rows
    for (int i = tid; i < (t1 - t0) * ncol; i += NTH)
      a.y[(long)(t0 + i / ncol) * H * P + h * P + c0 + i % ncol] = 0.f;
    return;
  }
  float* sp = a.state + ((long)slot * H + h) * N * P + c0;
  const bool fresh = a.positions[t0] == 0;
  // this wave's state tiles: column tile ct, row tiles (wave / 4) + 2 n
  const int ct = wave & 3, dt0 = wave >> 2;
  const int ndt = N >> 4;
  f32x4 sacc[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int dt = dt0 + 2 * n, c = ct * 16 + fr;
    sacc[n] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (dt < ndt) {
      if (!fresh && c < ncol) {
#pragma unroll
        for (int r = 0; r < 4; ++r) sacc[n][r] = sp[(long)(dt * 16 + 4 * q + r) * P + c];
      }
      *reinterpret_cast<f32x4*>(St + (ct * 16 + fr) * ldq + dt * 16 + 4 * q) = sacc[n];
    }
  }
  const int up = N >> 3;                   // staging units of a row: eight elements of B and C
  constexpr int MAXU = (C * NT * 4 + NTH - 1) / NTH;
  constexpr int VU = C * (CW / 4) / NTH;
  Row8<S> pq[MAXU], pk[MAXU];
  f32x4 pv[VU];
  float pdt = 0.f;
  const S* xr = (const S*)a.xc;
  const int voff = h * P + c0, koff = H * P + g * N, qoff = koff + G * N;
  const float bias = a.dt_bias[h], rate = a.rate[h], skip = a.skip[h];
  auto load = [&](int tc) {
    const int n = min(C, t1 - tc);
#pragma unroll
    for (int u = 0; u < MAXU; ++u) {
      const int it = tid + u * NTH;
      const int r = it / up, k = it - r * up;
      if (r < n) {
        const S* p = xr + (long)(tc + r) * a.ldx + 8 * k;
        pq[u].load(p + qoff);
        pk[u].load(p + koff);
      }
    }
#pragma unroll
    for (int u = 0; u < VU; ++u) {
      // 16 tokens x 4 quads a wave: short pieces of a row, conflict-light transposed stores
      const int blk = wave + 8 * u, t = (blk & (C / 16 - 1)) * 16 + fr;
      const int c = (blk / (C / 16)) * 16 + q * 4;
      pv[u] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (t < n && c < ncol) pv[u] = load4(xr + (long)(tc + t) * a.ldx + voff + c);
    }
    if (wave == 0) pdt = lane < n ? a.dt[(long)(tc + lane) * a.ldt + h] : 0.f;
  };
  auto stage = [&](int n) {
    const int rows = (n + 15) & ~15;
#pragma unroll
    for (int u = 0; u < MAXU; ++u) {
      const int it = tid + u * NTH;
      const int r = it / up, k = it - r * up;
      if (r >= rows) continue;
      f32x4 q0 = {0.f, 0.f, 0.f, 0.f}, q1 = q0, k0 = q0, k1 = q0;
      if (r < n) { pq[u].get(q0, q1); pk[u].get(k0, k1); }
      *reinterpret_cast<f32x4*>(Qs + r * ldq + 8 * k) = q0;
      *reinterpret_cast<f32x4*>(Qs + r * ldq + 8 * k + 4) = q1;
      *reinterpret_cast<f32x4*>(Ks + r * ldq + 8 * k) = k0;
      *reinterpret_cast<f32x4*>(Ks + r * ldq + 8 * k + 4) = k1;
    }
#pragma unroll
    for (int u = 0; u < VU; ++u) {
      const int blk = wave + 8 * u, t = (blk & (C / 16 - 1)) * 16 + fr;
      const int c = (blk / (C / 16)) * 16 + q * 4;
#pragma unroll
      for (int i = 0; i < 4; ++i) Vt[(c + i) * ldc + t] = pv[u][i];
    }
    if (wave == 0) {                       // a token a lane: step size, summed log decays
      const float st = lane < n ? softplus32(pdt + bias) : 0.f;
      double L = -(double)rate * (double)st;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const double v = __shfl_up(L, o, 64);
        if (lane >= o) L += v;
      }
      const double Ln = __shfl(L, 63, 64);
      if (lane < C) {
        const float hi = (float)L;
        lh[lane] = hi;
        ll[lane] = (float)(L - (double)hi);
        sz[lane] = st;
        eL[lane] = expf(hi);
        ew[lane] = st * expf((float)(Ln - L));
        if (lane == 0) en[0] = expf((float)Ln);
      }
    }
  };
  load(t0);
  for (int tc = t0; tc < t1; tc += C) {
    const int n = min(C, t1 - tc), nt = (n + 15) >> 4;
    __syncthreads();                       // the previous chunk is done with the LDS rows
    stage(n);
    __syncthreads();
    if (tc + C < t1) load(tc + C);         // in flight during the products
    // ---- P^T tiles (input rows, query columns), j <= i
    for (int tile = wave; tile < nt * (nt + 1) / 2; tile += 8) {
      int it = 0;
      while ((it + 1) * (it + 2) / 2 <= tile) ++it;
      const int jt = tile - it * (it + 1) / 2;
      const float* kp = Ks + (jt * 16 + fr) * ldq + 4 * q;
      const float* qp = Qs + (it * 16 + fr) * ldq + 4 * q;
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
      for (int x = 0; x < N; x += 16) {
        const f32x4 kf = *reinterpret_cast<const f32x4*>(kp + x);
        const f32x4 qf = *reinterpret_cast<const f32x4*>(qp + x);
#pragma unroll
        for (int i = 0; i < 4; ++i)
          acc = __builtin_amdgcn_mfma_f32_16x16x4f32(kf[i], qf[i], acc, 0, 0, 0);
      }
      const int i = it * 16 + fr, j = jt * 16 + 4 * q;
      const float hi = lh[i], lo = ll[i];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float e = expf(fminf((hi - lh[j + r]) + (lo - ll[j + r]), 0.f));
        acc[r] = j + r <= i ? acc[r] * (sz[j + r] * e) : 0.f;
        if (j + r == i) acc[r] += skip;
      }
      *reinterpret_cast<f32x4*>(Ps + i * ldc + j) = acc;
    }
    // ---- read-out of the state before the chunk, Y^T tiles (state columns, token columns):
    // this wave's column tile for tokens of row tiles dt0 and (chunk of four) 3 - dt0
    f32x4 oacc[C / 32];
#pragma unroll
    for (int m = 0; m < C / 32; ++m) oacc[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    {
      const float* vp = St + (ct * 16 + fr) * ldq + 4 * q;
      const float* qp = Qs + fr * ldq + 4 * q;
#pragma unroll 4
      for (int x = 0; x < N; x += 16) {
        const f32x4 sf = *reinterpret_cast<const f32x4*>(vp + x);
#pragma unroll
        for (int m = 0; m < C / 32; ++m) {
          const int it = m == 0 ? dt0 : 3 - dt0;
          if (it >= nt) continue;
          const f32x4 qf = *reinterpret_cast<const f32x4*>(qp + it * 16 * ldq + x);
#pragma unroll
          for (int i = 0; i < 4; ++i)
            oacc[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(sf[i], qf[i], oacc[m], 0, 0, 0);
        }
      }
#pragma unroll
      for (int m = 0; m < C / 32; ++m) {
        const int it = m == 0 ? dt0 : 3 - dt0;
        if (it < nt) oacc[m] *= eL[it * 16 + fr];
      }
    }
    // ---- the state after the chunk: input columns x decayed x
    f32x4 vf[C / 16];
#pragma unroll
    for (int jt = 0; jt < C / 16; ++jt) {
      if (jt >= nt) continue;
      vf[jt] = *reinterpret_cast<const f32x4*>(Vt + (ct * 16 + fr) * ldc + jt * 16 + 4 * q);
      vf[jt] *= *reinterpret_cast<const f32x4*>(ew + jt * 16 + 4 * q);
    }
    const float an = en[0];
#pragma unroll
    for (int m = 0; m < NT; ++m) {
      const int dt = dt0 + 2 * m;
      if (dt >= ndt) continue;
      sacc[m] *= an;
#pragma unroll
      for (int jt = 0; jt < C / 16; ++jt) {
        if (jt >= nt) continue;
        const float* kp = Ks + (jt * 16 + 4 * q) * ldq + dt * 16 + fr;
#pragma unroll
        for (int i = 0; i < 4; ++i)
          sacc[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(kp[i * ldq], vf[jt][i], sacc[m], 0, 0, 0);
      }
    }
    __syncthreads();                       // P complete; every read of the old state is done
#pragma unroll
    for (int m = 0; m < NT; ++m) {
      const int dt = dt0 + 2 * m;
      if (dt < ndt)
        *reinterpret_cast<f32x4*>(St + (ct * 16 + fr) * ldq + dt * 16 + 4 * q) = sacc[m];
    }
    // ---- Y += P . x
#pragma unroll
    for (int m = 0; m < C / 32; ++m) {
      const int it = m == 0 ? dt0 : 3 - dt0;
      if (it >= nt) continue;
      const float* vp = Vt + (ct * 16 + fr) * ldc + 4 * q;
      const float* pp = Ps + (it * 16 + fr) * ldc + 4 * q;
      for (int x = 0; x <= it * 16; x += 16) {
        const f32x4 vv = *reinterpret_cast<const f32x4*>(vp + x);
        const f32x4 pf = *reinterpret_cast<const f32x4*>(pp + x);
#pragma unroll
        for (int i = 0; i < 4; ++i)
          oacc[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(vv[i], pf[i], oacc[m], 0, 0, 0);
      }
      // lane: token it*16 + fr, columns ct*16 + 4q .. +3
      const int tok = it * 16 + fr, c = ct * 16 + 4 * q;
      if (tok < n && c < ncol)
        *reinterpret_cast<f32x4*>(a.y + (long)(tc + tok) * H * P + h * P + c0 + c) = oacc[m];
    }
  }
#pragma unroll
  for (int m = 0; m < NT; ++m) {
    const int dt = dt0 + 2 * m, c = ct * 16 + fr;
    if (dt < ndt && c < ncol) {
#pragma unroll
      for (int r = 0; r < 4; ++r) sp[(long)(dt * 16 + 4 * q + r) * P + c] = sacc[m][r];
    }
  }
}

template <typename S, int C, int NT, int D>
int launch_chunks(const SsdArgs& a, int num_seqs, hipStream_t st) {
  const size_t sh = ((size_t)2 * C * (a.N + PAD) + (size_t)(CW + C) * (C + PAD) +
                     (size_t)CW * (a.N + PAD) + 5 * C + 4) * 4;
  if (sh > 160 * 1024) return (int)hipErrorInvalidValue;
  if (sh > 48 * 1024) {
    hipError_t e = hipFuncSetAttribute((const void*)ssd_chunk_kernel<S, C, NT, D>,
                                       hipFuncAttributeMaxDynamicSharedMemorySize, (int)sh);
    if (e != hipSuccess) return (int)e;
  }
  dim3 grid(a.H, num_seqs, (a.P + CW - 1) / CW);
  ssd_chunk_kernel<S, C, NT, D><<<grid, NTH, sh, st>>>(a);
  DLI_RETURN_LAUNCH();
}

template <typename S>
int launch_chunks_any(const SsdArgs& a, int num_seqs, hipStream_t st) {
  if (a.N == 64) return launch_chunks<S, 64, 2, 64>(a, num_seqs, st);
  if (a.N == 128) return launch_chunks<S, 64, 4, 128>(a, num_seqs, st);
  if (a.N == 256) return launch_chunks<S, 32, 8, 256>(a, num_seqs, st);
  if (a.N <= 32) return launch_chunks<S, 64, 1, 0>(a, num_seqs, st);
  if (a.N <= 64) return launch_chunks<S, 64, 2, 0>(a, num_seqs, st);
  if (a.N <= 128) return launch_chunks<S, 64, 4, 0>(a, num_seqs, st);
  return launch_chunks<S, 32, 8, 0>(a, num_seqs, st);
}

// ------------------------------------------------------------------------------ single tokens
struct StepArgs {
  const float* u; int ldu;                 // x | B | C | dt before the filter
  const float* w; const float* b; int taps;
  const float* dt_bias; const float* rate; const float* skip;
  float* state; float* ring;
  const int* slots; const int* cu; const int* positions;
  float* y;
  int H, N, P, G;
};

// A workgroup per (head, sequence). Thread = (column quad cq of QP, row group rg of RG = 256 / QP);
// its R = ceil(N / RG) state quads stream through registers, all in flight at once. Every head
// of a group filters the group's B and C for itself; the group's first head stores their inputs.
template <int R, int TAPS>
__global__ void __launch_bounds__(256, R >= 32 ? 2 : 4) ssd_step_kernel(StepArgs a, int qp_log2) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int H = a.H, N = a.N, P = a.P, G = a.G;
  const int QP = 1 << qp_log2, RG = 256 >> qp_log2;
  float* xs = sm;                          // [P]
  float* bs = xs + P;                      // [N]
  float* cs = bs + N;                      // [N]
  float* ov = sm + ((P + 2 * N + 3) & ~3); // [RG][4 QP] partial read-outs
  const int h = blockIdx.x, s = blockIdx.y;
  const int t = a.cu[s];
  if (a.cu[s + 1] <= t) return;
  const int tid = threadIdx.x, cq = tid & (QP - 1), rg = tid >> qp_log2;
  const int slot = a.slots[s];
  const bool col = 4 * cq < P;
  float* yp = a.y + (long)t * H * P + h * P + 4 * cq;
  if (slot < 0) {                          // padding rows of a captured step
    if (col && rg == 0) *reinterpret_cast<f32x4*>(yp) = f32x4{0.f, 0.f, 0.f, 0.f};
    return;
  }
  const int p = a.positions[t];
  const int rep = H / G, g = h / rep, ch = H * P + 2 * G * N, ne = P + 2 * N;
  const int taps = TAPS ? TAPS : a.taps;
  const float* row = a.u + (long)t * a.ldu;
  float* ring = a.ring + (long)slot * taps * ch;
  const auto channel = [&](int e) {        // of this head's x, then its group's B, then its C
    return e < P ? h * P + e : e < P + N ? H * P + g * N + (e - P) : H * P + (G + g) * N + (e - P - N);
  };
  // the filter's inputs (two elements a thread at most sizes) are on their way before the state's
  constexpr int E = TAPS ? 2 : 1, KT = TAPS ? TAPS : 1;
  float in[E][KT], wt[E][KT], bias[E];
#pragma unroll
  for (int u = 0; u < E; ++u) {
    const int e = tid + 256 * u;
    if (TAPS == 0 || e >= ne) continue;
    const int c = channel(e);
    bias[u] = a.b[c];
    in[u][0] = row[c];
#pragma unroll
    for (int k = 1; k < KT; ++k)
      in[u][k] = k <= p ? ring[(long)((p - k) % KT) * ch + c] : 0.f;
#pragma unroll
    for (int k = 0; k < KT; ++k) wt[u][k] = a.w[(long)c * KT + KT - 1 - k];
  }
  const float zdt = row[ch + h] + a.dt_bias[h], rate = a.rate[h];
  float* sp = a.state + ((long)slot * H + h) * N * P + 4 * cq;
  f32x4 S[R];
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int r = rg + i * RG;
    S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (p != 0 && col && r < N) S[i] = *reinterpret_cast<const f32x4*>(sp + (long)r * P);
  }
#pragma unroll
  for (int u = 0; u < E; ++u) {
    const int e = tid + 256 * u;
    if (TAPS == 0 || e >= ne) continue;
    float acc = bias[u];
#pragma unroll
    for (int k = 0; k < KT; ++k) acc += wt[u][k] * in[u][k];
    if (e < P || h == g * rep) ring[(long)(p % KT) * ch + channel(e)] = in[u][0];
    sm[e] = silu32(acc);
  }
#pragma unroll 1
  for (int e = tid + (TAPS ? 256 * E : 0); e < ne; e += 256) {
    const int c = channel(e);
    const float cur = row[c];
    const float* w = a.w + (long)c * taps;
    float acc = a.b[c] + w[taps - 1] * cur;
    for (int k = 1; k < taps && k <= p; ++k)
      acc += w[taps - 1 - k] * ring[(long)((p - k) % taps) * ch + c];
    if (e < P || h == g * rep) ring[(long)(p % taps) * ch + c] = cur;
    sm[e] = silu32(acc);
  }
  const float st = softplus32(zdt);
  const float dec = expf(-rate * st);
  __syncthreads();
  f32x4 x = {0.f, 0.f, 0.f, 0.f};
  if (col) x = *reinterpret_cast<const f32x4*>(xs + 4 * cq);
  const f32x4 sx = st * x;
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int r = rg + i * RG;
    if (r < N) {
      S[i] = dec * S[i] + bs[r] * sx;
      o += cs[r] * S[i];
      if (col) *reinterpret_cast<f32x4*>(sp + (long)r * P) = S[i];
    }
  }
  *reinterpret_cast<f32x4*>(ov + (rg * QP + cq) * 4) = o;
  __syncthreads();
  if (rg == 0 && col) {
    o = a.skip[h] * x;
#pragma unroll 4
    for (int k = 0; k < RG; ++k) o += *reinterpret_cast<const f32x4*>(ov + (k * QP + cq) * 4);
    *reinterpret_cast<f32x4*>(yp) = o;
  }
}

}  // namespace

// ring [slots, taps, ch]; u [T, >= ch] with row stride ldu; out [T, ch] in the storage type dt
extern "C" int dli_ssd_conv(const float* u, int ldu, const float* w, const float* b, int taps,
                            float* ring, const int* slots, const int* cu, const int* positions,
                            void* out, int num_seqs, int max_seqlen, int ch, int dt,
                            hipStream_t st) {
  if (num_seqs <= 0 || max_seqlen <= 0) return 0;
  if (ch < 1 || taps < 1 || num_seqs > 65535 || ring == nullptr || slots == nullptr ||
      out == nullptr || ldu < ch || (dt != 0 && dt != 1))
    return (int)hipErrorInvalidValue;
  const int tb = taps > 33 ? taps - 1 : 32;        // a block's past lies inside the block before it
  ConvArgs a{u, ldu, w, b, taps, ring, slots, cu, positions, out, ch, tb};
  const bool v4 = ch % 4 == 0 && ldu % 4 == 0 &&
                  ((uintptr_t)u | (uintptr_t)ring | (uintptr_t)out) % 16 == 0;
  const int per = 256 * (v4 ? 4 : 1);
  dim3 grid((max_seqlen + tb - 1) / tb, num_seqs, (ch + per - 1) / per);
#define CONV_TAPS(S, V)                                                        \
  switch (taps) {                                                              \
    case 2: ssd_conv_kernel<S, V, 2><<<grid, 256, 0, st>>>(a); break;          \
    case 3: ssd_conv_kernel<S, V, 3><<<grid, 256, 0, st>>>(a); break;          \
    case 4: ssd_conv_kernel<S, V, 4><<<grid, 256, 0, st>>>(a); break;          \
    default: ssd_conv_kernel<S, V, 0><<<grid, 256, 0, st>>>(a); break;         \
  }
  if (dt == 0) { if (v4) { CONV_TAPS(u16, 4) } else { CONV_TAPS(u16, 1) } }
  else { if (v4) { CONV_TAPS(float, 4) } else { CONV_TAPS(float, 1) } }
#undef CONV_TAPS
  DLI_RETURN_LAUNCH();
}

// N a multiple of 16 up to 256, P of 4 (bf16 rows: of 8); rows 16-byte aligned
extern "C" int dli_ssd_chunks(const void* xc, int ldx, const float* dts, int ldt,
                              const float* dt_bias, const float* rate, const float* skip,
                              float* state, const int* slots, const int* cu, const int* positions,
                              float* y, int num_seqs, int H, int N, int P, int G, int dt,
                              hipStream_t st) {
  if (num_seqs <= 0) return 0;
  const int al = dt == 0 ? 8 : 4;
  if (H < 1 || G < 1 || H % G || N < 16 || N % 16 || N > 256 || P < 1 || P % al || ldx % al ||
      ldx < H * P + 2 * G * N || num_seqs > 65535 || (dt != 0 && dt != 1) || state == nullptr ||
      slots == nullptr || ((uintptr_t)xc | (uintptr_t)y) % 16)
    return (int)hipErrorInvalidValue;
  SsdArgs a{xc, ldx, dts, ldt, dt_bias, rate, skip, state, slots, cu, positions, y, H, N, P, G};
  return dt == 0 ? launch_chunks_any<u16>(a, num_seqs, st) : launch_chunks_any<float>(a, num_seqs, st);
}

// one token a sequence; hipErrorNotSupported for sizes it does not take
extern "C" int dli_ssd_step(const float* u, int ldu, const float* w, const float* b, int taps,
                            const float* dt_bias, const float* rate, const float* skip,
                            float* state, float* ring, const int* slots, const int* cu,
                            const int* positions, float* y, int num_seqs, int H, int N, int P,
                            int G, hipStream_t st) {
  if (num_seqs <= 0) return 0;
  if (H < 1 || G < 1 || H % G || N < 1 || P < 1 || taps < 1 || num_seqs > 65535 ||
      state == nullptr || ring == nullptr || slots == nullptr || ldu < H * P + 2 * G * N + H)
    return (int)hipErrorInvalidValue;
  int lg = 0;
  while ((4 << lg) < P) ++lg;              // column quads, rounded up to a power of two
  if (P % 4 || lg > 8 || ((uintptr_t)state | (uintptr_t)y) % 16) return (int)hipErrorNotSupported;
  const int RG = 256 >> lg, R = (N + RG - 1) / RG;
  const size_t sh = ((size_t)((P + 2 * N + 3) & ~3) + 1024) * 4;
  if (R > 32 || sh > 48 * 1024) return (int)hipErrorNotSupported;
  StepArgs a{u, ldu, w, b, taps, dt_bias, rate, skip, state, ring, slots, cu, positions, y, H, N, P, G};
  dim3 grid(H, num_seqs);
#define STEP_LAUNCH(RR)                                                              \
  do {                                                                               \
    if (taps == 4) ssd_step_kernel<RR, 4><<<grid, 256, sh, st>>>(a, lg);             \
    else ssd_step_kernel<RR, 0><<<grid, 256, sh, st>>>(a, lg);                       \
  } while (0)
  if (R <= 1) STEP_LAUNCH(1);
  else if (R <= 4) STEP_LAUNCH(4);
  else if (R <= 16) STEP_LAUNCH(16);
  else STEP_LAUNCH(32);
#undef STEP_LAUNCH
  DLI_RETURN_LAUNCH();
}
