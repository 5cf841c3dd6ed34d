// Retention (ops.hybrid.retention): linear attention with one fixed decay a per head over
// per-sequence fp32 state slots S [slots, H, d, dv],
//     S_t = a S_{t-1} + k_t v_t^T,      o_t = S_t^T q_t,
// q and k rotated (the first `rot` dims of every head, dimension i with i + rot/2), k times
// d^(-1/2); o_t is divided by its RMS per head and multiplied by silu(gate_t).
//
// Chunk form (portions). A chunk of n <= C tokens that starts from state S_0 obeys
//     o_i = a^(i+1) S_0^T q_i + sum_{j <= i} a^(i-j) (k_j . q_i) v_j          i = 0 .. n-1
//     S_n = a^n S_0 + sum_j a^(n-1-j) k_j v_j^T
// four matrix products, run on the fp32 matrix cores (v_mfma_f32_16x16x4_f32: everything that
// enters the recurrence stays fp32, for both storage types). One workgroup of 8 waves per (head,
// sequence, block of 64 state columns) walks the sequence's chunks: the state block lives in the
// accumulators of product 4 and, transposed, in LDS as an operand of the read-out; the next
// chunk's projections are in flight in registers while a chunk is computed.
//
// The summation index of an MFMA may be permuted as long as both operands agree, so a lane
// takes four consecutive k with one 16-byte LDS read and feeds four MFMAs with them: rows are
// padded by 8 floats, which spreads every 16-lane group over all banks.
//
// With more than one column block no workgroup sees a whole head: o_t leaves in fp32 (`raw`)
// and the caller norms and gates it. Single tokens (decode steps) and shapes this form does
// not take run the walk of recurrent_scalar.hip.
#include "common.h"

// recurrent_scalar.hip
int retention_walk(const float* proj, int ldp, const float* table, int rot, const float* decay_pow,
                   int ldd, float eps, float* state, const int* slots, const int* cu,
                   const int* positions, void* out, int ldo, int num_seqs, int H, int d, int dv,
                   int cw, float* raw, int dt, hipStream_t st);

namespace {

template <typename S> __device__ __forceinline__ void stf4(S* p, f32x4 v);
template <> __device__ __forceinline__ void stf4<float>(float* p, f32x4 v) {
  *reinterpret_cast<f32x4*>(p) = v;
}
template <> __device__ __forceinline__ void stf4<u16>(u16* p, f32x4 v) {
  uint2 pk;
  pk.x = pack2bf(v[0], v[1]);
  pk.y = pack2bf(v[2], v[3]);
  *reinterpret_cast<uint2*>(p) = pk;
}

constexpr int CW = 64;            // state columns of a workgroup
constexpr int NTH = 512;          // 8 waves
constexpr int PAD = 8;

struct RetentionArgs {
  const float* proj; int ldp;
  const float* table; int rot;     // [T, rot] cosines | sines
  const float* pw; int ldw;        // [H][ldw] powers of the decay
  float kscale, eps;
  float* state;
  const int* slots; const int* cu; const int* positions;
  void* out; int ldo;              // [T, H*dv]
  float* raw;                      // several column blocks: o_t, fp32 [T, H*dv]
  int H, d, dv;
};

// C tokens a chunk; NT: 16-row state tiles a wave accumulates (d <= 32 NT)
template <typename S, int C, int NT>
__global__ void __launch_bounds__(NTH) retention_chunk_kernel(RetentionArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int d = a.d, dv = a.dv, H = a.H;
  const int ldq = d + PAD;
  constexpr int ldc = C + PAD;
  float* Qs = sm;                          // [C][ldq] rotated queries
  float* Ks = Qs + C * ldq;                // [C][ldq] rotated, scaled keys
  float* Vt = Ks + C * ldq;                // [CW][ldc] values, transposed
  float* Ps = Vt + CW * ldc;               // [C][ldc] decayed key-query products (query rows)
  float* St = Ps + C * ldc;                // [CW][ldq] the state before the chunk, transposed
  float* pw = St + CW * ldq;               // [C + 1] (padded to C + 4)
  float* red = pw + C + 4;                 // [C][4] partial sums of squares
  const int h = blockIdx.x, s = blockIdx.y, c0 = blockIdx.z * CW;
  const int ncol = min(CW, dv - c0);
  const int slot = a.slots[s], t0 = a.cu[s], t1 = a.cu[s + 1];
  if (t1 <= t0) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int fr = lane & 15, q = lane >> 4;
  if (slot < 0) {                          // padding rows
    for (int i = tid; i < (t1 - t0) * ncol; i += NTH) {
      const long o = (long)(t0 + i / ncol);
      const int c = h * dv + c0 + i % ncol;
      if (a.raw != nullptr) a.raw[o * H * dv + c] = 0.f;
      else if (sizeof(S) == 2) ((u16*)a.out)[o * a.ldo + c] = 0;
      else ((float*)a.out)[o * a.ldo + c] = 0.f;
    }
    return;
  }
  for (int i = tid; i <= C; i += NTH) pw[i] = a.pw[(long)h * a.ldw + i];
  float* sp = a.state + ((long)slot * H + h) * d * dv + c0;
  const bool fresh = a.positions[t0] == 0;
  // this wave's state tiles: column tile ct, row tiles (wave / 4) + 2 n
  const int ct = wave & 3, dt0 = wave >> 2;
  const int ndt = d >> 4;
  f32x4 sacc[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int dt = dt0 + 2 * n, c = ct * 16 + fr;
    sacc[n] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (dt < ndt) {
      if (!fresh && c < ncol) {
#pragma unroll
        for (int r = 0; r < 4; ++r) sacc[n][r] = sp[(long)(dt * 16 + 4 * q + r) * dv + c];
      }
      *reinterpret_cast<f32x4*>(St + (ct * 16 + fr) * ldq + dt * 16 + 4 * q) = sacc[n];
    }
  }
  // staging: a unit is a pair of rotated quads (c, c + rot/2) or one quad that passes
  const int hr = a.rot >> 1, rq = hr >> 2, up = rq + ((d - a.rot) >> 2);
  constexpr int MAXU = (C * NT * 8 + NTH - 1) / NTH;
  constexpr int VU = C * (CW / 4) / NTH;
  f32x4 pq[MAXU][2], pk[MAXU][2], tb[MAXU][2], pv[VU];
  const int voff = 2 * H * d + h * dv + c0;
  auto load = [&](int tc) {
    const int n = min(C, t1 - tc);
#pragma unroll
    for (int u = 0; u < MAXU; ++u) {
      const int it = tid + u * NTH;
      const int r = it / up, k = it - r * up;
      if (r < n) {
        const bool pair = k < rq;
        const int c = pair ? 4 * k : a.rot + 4 * (k - rq);
        const float* p = a.proj + (long)(tc + r) * a.ldp + h * d + c;
        pq[u][0] = *reinterpret_cast<const f32x4*>(p);
        pk[u][0] = *reinterpret_cast<const f32x4*>(p + H * d);
        if (pair) {
          pq[u][1] = *reinterpret_cast<const f32x4*>(p + hr);
          pk[u][1] = *reinterpret_cast<const f32x4*>(p + H * d + hr);
          const float* tp = a.table + (long)(tc + r) * a.rot + c;
          tb[u][0] = *reinterpret_cast<const f32x4*>(tp);
          tb[u][1] = *reinterpret_cast<const f32x4*>(tp + hr);
        }
      }
    }
#pragma unroll
    for (int u = 0; u < VU; ++u) {
      // 16 tokens x 4 quads a wave: 64-byte pieces of a row, conflict-light transposed stores
      const int blk = wave + 8 * u, t = (blk & (C / 16 - 1)) * 16 + fr;
      const int c = (blk / (C / 16)) * 16 + q * 4;
      pv[u] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (t < n && c < ncol)
        pv[u] = *reinterpret_cast<const f32x4*>(a.proj + (long)(tc + t) * a.ldp + voff + c);
    }
  };
  auto stage = [&](int n) {
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    const int rows = (n + 15) & ~15;
#pragma unroll
    for (int u = 0; u < MAXU; ++u) {
      const int it = tid + u * NTH;
      const int r = it / up, k = it - r * up;
      if (r >= rows) continue;
      const bool pair = k < rq;
      const int c = pair ? 4 * k : a.rot + 4 * (k - rq);
      float* qd = Qs + r * ldq + c;
      float* kd = Ks + r * ldq + c;
      if (r >= n) {
        *reinterpret_cast<f32x4*>(qd) = zero;
        *reinterpret_cast<f32x4*>(kd) = zero;
        if (pair) {
          *reinterpret_cast<f32x4*>(qd + hr) = zero;
          *reinterpret_cast<f32x4*>(kd + hr) = zero;
        }
      } else if (pair) {
        const f32x4 cs = tb[u][0], sn = tb[u][1];
        *reinterpret_cast<f32x4*>(qd) = pq[u][0] * cs - pq[u][1] * sn;
        *reinterpret_cast<f32x4*>(qd + hr) = pq[u][1] * cs + pq[u][0] * sn;
        *reinterpret_cast<f32x4*>(kd) = (pk[u][0] * cs - pk[u][1] * sn) * a.kscale;
        *reinterpret_cast<f32x4*>(kd + hr) = (pk[u][1] * cs + pk[u][0] * sn) * a.kscale;
      } else {
        *reinterpret_cast<f32x4*>(qd) = pq[u][0];
        *reinterpret_cast<f32x4*>(kd) = pk[u][0] * a.kscale;
      }
    }
#pragma unroll
    for (int u = 0; u < VU; ++u) {
      const int blk = wave + 8 * u, t = (blk & (C / 16 - 1)) * 16 + fr;
      const int c = (blk / (C / 16)) * 16 + q * 4;
#pragma unroll
      for (int i = 0; i < 4; ++i) Vt[(c + i) * ldc + t] = pv[u][i];
    }
  };
  load(t0);
  for (int tc = t0; tc < t1; tc += C) {
    const int n = min(C, t1 - tc), nt = (n + 15) >> 4;
    __syncthreads();                       // the previous chunk is done with the LDS rows
    stage(n);
    __syncthreads();
    if (tc + C < t1) load(tc + C);         // in flight during the products
    // ---- P^T tiles (key rows, query columns): a^(i-j) k_j . q_i for j <= i
    for (int tile = wave; tile < nt * (nt + 1) / 2; tile += 8) {
      int it = 0;
      while ((it + 1) * (it + 2) / 2 <= tile) ++it;
      const int jt = tile - it * (it + 1) / 2;
      const float* kp = Ks + (jt * 16 + fr) * ldq + 4 * q;
      const float* qp = Qs + (it * 16 + fr) * ldq + 4 * q;
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
      for (int x = 0; x < d; x += 16) {
        const f32x4 kf = *reinterpret_cast<const f32x4*>(kp + x);
        const f32x4 qf = *reinterpret_cast<const f32x4*>(qp + x);
#pragma unroll
        for (int i = 0; i < 4; ++i)
          acc = __builtin_amdgcn_mfma_f32_16x16x4f32(kf[i], qf[i], acc, 0, 0, 0);
      }
      const int i = it * 16 + fr, j = jt * 16 + 4 * q;
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[r] = j + r <= i ? acc[r] * pw[max(i - j - r, 0)] : 0.f;
      *reinterpret_cast<f32x4*>(Ps + i * ldc + j) = acc;
    }
    // ---- read-out of the state before the chunk, O^T tiles (state columns, token columns):
    // this wave's column tile for tokens of row tiles dt0 and (chunk of four) 3 - dt0
    f32x4 oacc[C / 32];
#pragma unroll
    for (int m = 0; m < C / 32; ++m) {
      const int it = m == 0 ? dt0 : 3 - dt0;
      oacc[m] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (it >= nt) continue;
      const float* vp = St + (ct * 16 + fr) * ldq + 4 * q;
      const float* qp = Qs + (it * 16 + fr) * ldq + 4 * q;
      for (int x = 0; x < d; x += 16) {
        const f32x4 sf = *reinterpret_cast<const f32x4*>(vp + x);
        const f32x4 qf = *reinterpret_cast<const f32x4*>(qp + x);
#pragma unroll
        for (int i = 0; i < 4; ++i)
          oacc[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(sf[i], qf[i], oacc[m], 0, 0, 0);
      }
      oacc[m] *= pw[it * 16 + fr + 1];
    }
    // ---- the state after the chunk: key columns (dims) x decayed values
    f32x4 vf[C / 16];
#pragma unroll
    for (int jt = 0; jt < C / 16; ++jt) {
      if (jt >= nt) continue;
      vf[jt] = *reinterpret_cast<const f32x4*>(Vt + (ct * 16 + fr) * ldc + jt * 16 + 4 * q);
#pragma unroll
      for (int i = 0; i < 4; ++i) vf[jt][i] *= pw[max(n - 1 - (jt * 16 + 4 * q + i), 0)];
    }
    const float an = pw[n];
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
    // ---- O += P . V
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
      if (a.raw != nullptr) {
        if (tok < n && c < ncol)
          *reinterpret_cast<f32x4*>(a.raw + (long)(tc + tok) * H * dv + h * dv + c0 + c) = oacc[m];
      } else {
        float ss = (oacc[m][0] * oacc[m][0] + oacc[m][1] * oacc[m][1]) +
                   (oacc[m][2] * oacc[m][2] + oacc[m][3] * oacc[m][3]);
        ss += __shfl_xor(ss, 16, 64);
        ss += __shfl_xor(ss, 32, 64);
        if (q == 0) red[tok * 4 + ct] = ss;
      }
    }
    if (a.raw == nullptr) {                // one column block: the head's norm and gate here
      __syncthreads();
#pragma unroll
      for (int m = 0; m < C / 32; ++m) {
        const int it = m == 0 ? dt0 : 3 - dt0;
        const int tok = it * 16 + fr, c = ct * 16 + 4 * q;
        if (it >= nt || tok >= n || c >= ncol) continue;
        const f32x4 rr = *reinterpret_cast<const f32x4*>(red + tok * 4);
        const float rs = 1.f / sqrtf(((rr[0] + rr[1]) + (rr[2] + rr[3])) / (float)dv + a.eps);
        const long t = tc + tok;
        const f32x4 g = *reinterpret_cast<const f32x4*>(a.proj + t * a.ldp + 2 * H * d + H * dv +
                                                        h * dv + c0 + c);
        f32x4 o;
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] = oacc[m][i] * rs * (g[i] / (1.f + expf(-g[i])));
        stf4((S*)a.out + t * a.ldo + h * dv + c0 + c, o);
      }
    }
  }
#pragma unroll
  for (int m = 0; m < NT; ++m) {
    const int dt = dt0 + 2 * m, c = ct * 16 + fr;
    if (dt < ndt && c < ncol) {
#pragma unroll
      for (int r = 0; r < 4; ++r) sp[(long)(dt * 16 + 4 * q + r) * dv + c] = sacc[m][r];
    }
  }
}

template <typename S, int C, int NT>
int launch_chunks(const RetentionArgs& a, int num_seqs, hipStream_t st) {
  const size_t sh = ((size_t)2 * C * (a.d + PAD) + (size_t)(CW + C) * (C + PAD) +
                     (size_t)CW * (a.d + PAD) + C + 4 + C * 4) * 4;
  if (sh > 160 * 1024) return (int)hipErrorInvalidValue;
  if (sh > 48 * 1024) {
    hipError_t e = hipFuncSetAttribute((const void*)retention_chunk_kernel<S, C, NT>,
                                       hipFuncAttributeMaxDynamicSharedMemorySize, (int)sh);
    if (e != hipSuccess) return (int)e;
  }
  dim3 grid(a.H, num_seqs, (a.dv + CW - 1) / CW);
  retention_chunk_kernel<S, C, NT><<<grid, NTH, sh, st>>>(a);
  DLI_RETURN_LAUNCH();
}

template <typename S>
int launch_chunks_any(const RetentionArgs& a, int num_seqs, hipStream_t st) {
  if (a.d <= 32) return launch_chunks<S, 64, 1>(a, num_seqs, st);
  if (a.d <= 64) return launch_chunks<S, 64, 2>(a, num_seqs, st);
  if (a.d <= 128) return launch_chunks<S, 64, 4>(a, num_seqs, st);
  return launch_chunks<S, 32, 8>(a, num_seqs, st);
}

}  // namespace

// chunked != 0: the chunk form (column blocks of 64; d a multiple of 16 up to 256, dv of 4, rot
// of 8, 16-byte aligned rows); else the walk with column blocks of cw (0: one block). raw
// (fp32 [T, H*dv]) is given exactly when there are several column blocks.
extern "C" int dli_retention(const float* proj, int ldp, const float* table, int rot,
                             const float* decay_pow, int ldd, float kscale, float eps,
                             float* state, const int* slots, const int* cu, const int* positions,
                             void* out, int ldo, int num_seqs, int max_seqlen, int H, int d,
                             int dv, int cw, float* raw, int chunked, int dt, hipStream_t st) {
  if (num_seqs <= 0 || max_seqlen <= 0) return 0;
  if (H < 1 || d < 1 || dv < 1 || rot < 0 || (rot & 1) || rot > d || ldd < 65 || cw < 0 ||
      (cw > 0 && cw % 64) || (rot > 0 && table == nullptr) || state == nullptr ||
      slots == nullptr || decay_pow == nullptr || out == nullptr || (dt != 0 && dt != 1) ||
      num_seqs > 65535)
    return (int)hipErrorInvalidValue;
  if (!chunked) {
    if (cw == 0 || cw >= dv) cw = dv;
    if ((cw < dv) != (raw != nullptr)) return (int)hipErrorInvalidValue;
    return retention_walk(proj, ldp, table, rot, decay_pow, ldd, eps, state, slots, cu, positions,
                          out, ldo, num_seqs, H, d, dv, cw, raw, dt, st);
  }
  const uintptr_t mis = (uintptr_t)proj | (uintptr_t)table | (uintptr_t)out | (uintptr_t)raw;
  if (d % 16 || d > 256 || dv % 4 || rot % 8 || ldp % 4 || ldo % 4 || mis % 16 ||
      (dv > CW) != (raw != nullptr))
    return (int)hipErrorInvalidValue;
  RetentionArgs a{proj, ldp, table, rot, decay_pow, ldd, kscale, eps, state, slots, cu,
                  positions, out, ldo, raw, H, d, dv};
  return dt == 0 ? launch_chunks_any<u16>(a, num_seqs, st) : launch_chunks_any<float>(a, num_seqs, st);
}
