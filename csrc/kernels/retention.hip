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
// and the caller norms and gates it.
//
// Decode steps (one token a sequence) stream the state through registers, with rotation, norm
// and gate in the same launch. Shapes neither form takes, and portions of a few tokens, run the
// walk of recurrent_scalar.hip.
#include "common.h"

// recurrent_scalar.hip
int retention_walk(const float* proj, int ldp, const float* table, int rot, const float* decay_pow,
                   int ldd, float eps, float* state, const int* slots, const int* cu,
                   const int* positions, void* out, int ldo, int num_seqs, int H, int d, int dv,
                   int cw, float* raw, int dt, hipStream_t st);

namespace {

// four elements at index i of the output, bf16 (dt 0) or fp32 (dt 1)
__device__ __forceinline__ void store4(void* out, int dt, long i, f32x4 v) {
  if (dt == 0) {
    uint2 pk;
    pk.x = pack2bf(v[0], v[1]);
    pk.y = pack2bf(v[2], v[3]);
    *reinterpret_cast<uint2*>((u16*)out + i) = pk;
  } else {
    *reinterpret_cast<f32x4*>((float*)out + i) = v;
  }
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
  int H, d, dv, dt;
};

// C tokens a chunk; NT: 16-row state tiles a wave accumulates (d <= 32 NT); D: d when it is known
// at compile time (else 0)
template <int C, int NT, int D>
__global__ void __launch_bounds__(NTH) retention_chunk_kernel(RetentionArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int d = D ? D : a.d, dv = a.dv, H = a.H;
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
      else if (a.dt == 0) ((u16*)a.out)[o * a.ldo + c] = 0;
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
  // staging: a unit is two quads of a row, rotated partners (c, c + rot/2) or, past the rotated
  // dims, neighbours: d/8 units a row whatever rotates
  const int hr = a.rot >> 1, rq = hr >> 2, up = d >> 3;
  constexpr int MAXU = (C * NT * 4 + NTH - 1) / NTH;
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
        const int c = pair ? 4 * k : a.rot + 8 * (k - rq), c2 = pair ? c + hr : c + 4;
        const float* p = a.proj + (long)(tc + r) * a.ldp + h * d;
        pq[u][0] = *reinterpret_cast<const f32x4*>(p + c);
        pq[u][1] = *reinterpret_cast<const f32x4*>(p + c2);
        pk[u][0] = *reinterpret_cast<const f32x4*>(p + H * d + c);
        pk[u][1] = *reinterpret_cast<const f32x4*>(p + H * d + c2);
        if (pair) {
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
      const int c = pair ? 4 * k : a.rot + 8 * (k - rq), c2 = pair ? c + hr : c + 4;
      f32x4 q0 = zero, q1 = zero, k0 = zero, k1 = zero;
      if (r < n) {
        q0 = pq[u][0]; q1 = pq[u][1];
        k0 = pk[u][0]; k1 = pk[u][1];
        if (pair) {
          const f32x4 cs = tb[u][0], sn = tb[u][1];
          q0 = pq[u][0] * cs - pq[u][1] * sn;
          q1 = pq[u][1] * cs + pq[u][0] * sn;
          k0 = pk[u][0] * cs - pk[u][1] * sn;
          k1 = pk[u][1] * cs + pk[u][0] * sn;
        }
        k0 *= a.kscale;
        k1 *= a.kscale;
      }
      *reinterpret_cast<f32x4*>(Qs + r * ldq + c) = q0;
      *reinterpret_cast<f32x4*>(Qs + r * ldq + c2) = q1;
      *reinterpret_cast<f32x4*>(Ks + r * ldq + c) = k0;
      *reinterpret_cast<f32x4*>(Ks + r * ldq + c2) = k1;
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
#pragma unroll (D ? 4 : 1)
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
    for (int m = 0; m < C / 32; ++m) oacc[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    {
      const float* vp = St + (ct * 16 + fr) * ldq + 4 * q;
      const float* qp = Qs + fr * ldq + 4 * q;
#pragma unroll (D ? 4 : 1)
      for (int x = 0; x < d; x += 16) {
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
        if (it < nt) oacc[m] *= pw[it * 16 + fr + 1];
      }
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
        store4(a.out, a.dt, t * a.ldo + h * dv + c0 + c, o);
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

template <int C, int NT, int D>
int launch_chunks(const RetentionArgs& a, int num_seqs, hipStream_t st) {
  const size_t sh = ((size_t)2 * C * (a.d + PAD) + (size_t)(CW + C) * (C + PAD) +
                     (size_t)CW * (a.d + PAD) + C + 4 + C * 4) * 4;
  if (sh > 160 * 1024) return (int)hipErrorInvalidValue;
  if (sh > 48 * 1024) {
    hipError_t e = hipFuncSetAttribute((const void*)retention_chunk_kernel<C, NT, D>,
                                       hipFuncAttributeMaxDynamicSharedMemorySize, (int)sh);
    if (e != hipSuccess) return (int)e;
  }
  dim3 grid(a.H, num_seqs, (a.dv + CW - 1) / CW);
  retention_chunk_kernel<C, NT, D><<<grid, NTH, sh, st>>>(a);
  DLI_RETURN_LAUNCH();
}

int launch_chunks_any(const RetentionArgs& a, int num_seqs, hipStream_t st) {
  if (a.d == 64) return launch_chunks<64, 2, 64>(a, num_seqs, st);
  if (a.d == 128) return launch_chunks<64, 4, 128>(a, num_seqs, st);
  if (a.d == 256) return launch_chunks<32, 8, 256>(a, num_seqs, st);
  if (a.d <= 32) return launch_chunks<64, 1, 0>(a, num_seqs, st);
  if (a.d <= 64) return launch_chunks<64, 2, 0>(a, num_seqs, st);
  if (a.d <= 128) return launch_chunks<64, 4, 0>(a, num_seqs, st);
  return launch_chunks<32, 8, 0>(a, num_seqs, st);
}

// One token a sequence (decode steps): a workgroup per (head, sequence). Thread = (column quad
// cq of QP, row group rg of RG = 256 / QP); its R = ceil(d / RG) state quads stream through
// registers, all in flight at once: one read and one write per element.
template <int R>
__global__ void __launch_bounds__(256, R >= 32 ? 2 : 4) retention_step_kernel(RetentionArgs a, int qp_log2) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int d = a.d, dv = a.dv, H = a.H;
  const int QP = 1 << qp_log2, RG = 256 >> qp_log2;
  float* qs = sm;                          // [d], padded to a multiple of 4
  float* ks = qs + ((d + 3) & ~3);         // [d]
  float* ov = ks + ((d + 3) & ~3);         // [RG][4 QP] partial read-outs
  float* red = ov + RG * 4 * QP;           // [16]
  const int h = blockIdx.x, s = blockIdx.y;
  const int t = a.cu[s];
  if (a.cu[s + 1] <= t) return;
  const int tid = threadIdx.x, cq = tid & (QP - 1), rg = tid >> qp_log2;
  const int slot = a.slots[s];
  const long oi = (long)t * a.ldo + h * dv;
  const bool col = 4 * cq < dv;
  if (slot < 0) {                          // padding rows of a captured step
    if (col && rg == 0) store4(a.out, a.dt, oi + 4 * cq, f32x4{0.f, 0.f, 0.f, 0.f});
    return;
  }
  const bool fresh = a.positions[t] == 0;
  float* sp = a.state + ((long)slot * H + h) * d * dv + 4 * cq;
  f32x4 S[R];
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int r = rg + i * RG;
    S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (!fresh && col && r < d) S[i] = *reinterpret_cast<const f32x4*>(sp + (long)r * dv);
  }
  const float* row = a.proj + (long)t * a.ldp;
  f32x4 v = {0.f, 0.f, 0.f, 0.f};
  if (col) v = *reinterpret_cast<const f32x4*>(row + 2 * H * d + h * dv + 4 * cq);
  const int hr = a.rot >> 1;
  for (int i = tid; i < d; i += 256) {
    float q = row[h * d + i], k = row[H * d + h * d + i];
    if (i < a.rot) {
      const bool second = i >= hr;
      const int ci = second ? i - hr : i, pi = second ? i - hr : i + hr;
      const float* tb = a.table + (long)t * a.rot;
      const float cs = tb[ci], sn = second ? tb[hr + ci] : -tb[hr + ci];
      q = q * cs + row[h * d + pi] * sn;
      k = k * cs + row[H * d + h * d + pi] * sn;
    }
    qs[i] = q;
    ks[i] = k * a.kscale;
  }
  const float dec = a.pw[(long)h * a.ldw + 1];
  __syncthreads();
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int r = rg + i * RG;
    if (r < d) {
      S[i] = dec * S[i] + ks[r] * v;
      o += qs[r] * S[i];
      if (col) *reinterpret_cast<f32x4*>(sp + (long)r * dv) = S[i];
    }
  }
  *reinterpret_cast<f32x4*>(ov + (rg * QP + cq) * 4) = o;
  __syncthreads();
  float ss = 0.f;
  o = f32x4{0.f, 0.f, 0.f, 0.f};
  if (rg == 0) {
    for (int g = 0; g < RG; ++g) o += *reinterpret_cast<const f32x4*>(ov + (g * QP + cq) * 4);
    ss = (o[0] * o[0] + o[1] * o[1]) + (o[2] * o[2] + o[3] * o[3]);
  }
  ss = block_sum(ss, red);
  if (rg == 0 && col) {
    const float rs = 1.f / sqrtf(ss / (float)dv + a.eps);
    const f32x4 g = *reinterpret_cast<const f32x4*>(row + 2 * H * d + H * dv + h * dv + 4 * cq);
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] *= rs * (g[i] / (1.f + expf(-g[i])));
    store4(a.out, a.dt, oi + 4 * cq, o);
  }
}

int launch_step(const RetentionArgs& a, int num_seqs, hipStream_t st) {
  int lg = 0;
  while ((4 << lg) < a.dv) ++lg;           // column quads, rounded up to a power of two
  if (lg > 8) return (int)hipErrorNotSupported;
  const int RG = 256 >> lg, R = (a.d + RG - 1) / RG;
  const size_t sh = ((size_t)2 * ((a.d + 3) & ~3) + 1024 + 16) * 4;
  if (R > 32 || sh > 48 * 1024) return (int)hipErrorNotSupported;
  dim3 grid(a.H, num_seqs);
  if (R <= 1) retention_step_kernel<1><<<grid, 256, sh, st>>>(a, lg);
  else if (R <= 4) retention_step_kernel<4><<<grid, 256, sh, st>>>(a, lg);
  else if (R <= 16) retention_step_kernel<16><<<grid, 256, sh, st>>>(a, lg);
  else retention_step_kernel<32><<<grid, 256, sh, st>>>(a, lg);
  DLI_RETURN_LAUNCH();
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
  const uintptr_t mis = (uintptr_t)proj | (uintptr_t)table | (uintptr_t)out | (uintptr_t)raw |
                        (uintptr_t)state;
  const bool quads = dv % 4 == 0 && ldp % 4 == 0 && ldo % 4 == 0 && (H * d) % 2 == 0 &&
                     mis % 16 == 0;
  RetentionArgs a{proj, ldp, table, rot, decay_pow, ldd, kscale, eps, state, slots, cu,
                  positions, out, ldo, raw, H, d, dv, dt};
  if (!chunked) {
    if (max_seqlen == 1 && quads && raw == nullptr) {
      const int rc = launch_step(a, num_seqs, st);
      if (rc != (int)hipErrorNotSupported) return rc;
    }
    if (cw == 0 || cw >= dv) cw = dv;
    if ((cw < dv) != (raw != nullptr)) return (int)hipErrorInvalidValue;
    return retention_walk(proj, ldp, table, rot, decay_pow, ldd, eps, state, slots, cu, positions,
                          out, ldo, num_seqs, H, d, dv, cw, raw, dt, st);
  }
  if (d % 16 || d > 256 || !quads || rot % 8 || (dv > CW) != (raw != nullptr))
    return (int)hipErrorInvalidValue;
  return launch_chunks_any(a, num_seqs, st);
}
