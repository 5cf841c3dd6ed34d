// Grouped-query sliding-window attention with kept first tokens over token-major paged caches
// (ops.hybrid.window_attention: bf16, the key / value widths in SWA_WIDTHS, an optional elementwise
// gate on the output, no bias, mixing, head gate or sink — those run window_attention_mfma.hip).
// Position i sees j <= i with i - j < window or j < keep.
//
// The keys that a group of queries can see are at most two runs, [0, kf) and [lo, last], walked
// as one list: list index x is key x for x < kf and key x + skip from there on. Everything below
// tiles that list, so kept tokens cost what they are and nothing between them and the window is
// read.
//
//  * swa_prefill32  8 waves x 32 query rows of one head: v_mfma_f32_32x32x16_bf16 on swapped
//                   products (S^T = K . Q^T, O^T = V^T . P^T), so that a lane owns one query and
//                   the softmax is lane-local but for one exchange; K / V tiles of 64 keys by
//                   LDS-DMA into three buffers, one barrier a tile; the list's cache rows looked
//                   up once (LDS). The structure of attention_prefill.hip's long-prompt kernel.
//  * swa_prefill16  4 waves x 16 query rows: portions shorter than the above is worth
//  * swa_decode     one query token a sequence: a workgroup per (sequence, kv head, key split).
//                   Scores on the matrix cores with K rows straight from the cache (the heads
//                   of the group are the columns); the value sum in fp32 FMAs, a lane owning 8
//                   dims of every head of the group: at one row per head it is far below the
//                   time the bytes take, and V needs no transpose.
#include "common.h"

typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef short s16x8 __attribute__((ext_vector_type(8)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) void lds_void;
typedef const __attribute__((address_space(1))) void gbl_void;

namespace {

constexpr float LOG2E = 1.4426950408889634f;

struct SwaArgs {
  const u16* q; int ldq;
  const u16* k; long k_stride;         // cache rows
  const u16* v; long v_stride;
  u16* out; int ldo;
  const float* gate; int ldg;          // null, or [T, H*dv]: the output times its sigmoid
  const int* cu; const int* positions;
  const int* block_tables; int bt_stride; int block_size;
  int H, G, window, keep;
  float scale_log2;
  int table_cap;                       // prefill32: list entries that fit the LDS table
  int nsplit;                          // decode: key splits
  float* ws;                           // decode, nsplit > 1: [nsplit][S][H][2], [nsplit][S][H][HD]
};

// floats of the decode splits' (max, sum) pairs, in front of their partial sums
__host__ __device__ inline long stat_floats(int nsplit, int S, int H) {
  return ((long)nsplit * S * H * 2 + 3) & ~3L;
}

__device__ __forceinline__ float sigmoid32(float g) { return 1.f / (1.f + __expf(-g)); }

// the key list of queries at positions [first, last]
struct KeyList {
  int kf, skip, n;
  __device__ KeyList(int first, int last, int window, int keep) {
    const int lo = max(0, first - window + 1);
    kf = min(keep, lo);
    skip = lo - kf;
    n = last - skip + 1;
  }
  __device__ int key(int x) const { return x < kf ? x : x + skip; }
};

__device__ __forceinline__ float max3(float a, float b, float c) {
  return fmaxf(fmaxf(a, b), c);
}

constexpr int KT = 64;                 // keys a tile
constexpr int LROWS = 256;             // query rows of a long-form workgroup
constexpr float RESCALE_THR = 8.f;     // log2 units: the running max moves only by more than this

// One tile of rows (D wide) by LDS-DMA: 1-KiB pieces of two subtiles in a row, wave w of 8 takes
// pieces w, w + 8, ... The DMA writes lane-linearly, so each lane loads the logical chunk that
// lands at its place.
template <int D, typename RowOf>
__device__ __forceinline__ void stage_rows(const u16* src, long stride, char* dst, int x0, int wid,
                                           int lane, const RowOf& row_of) {
  constexpr int NP = D / 8;
#pragma unroll
  for (int j = 0; j < (NP + 7) / 8; ++j) {
    const int piece = wid + 8 * j;
    if (NP % 8 != 0 && piece >= NP) break;                     // wave-uniform
    const int b = piece * 1024 + lane * 16;
    const int rg = b / (D * 16), in = b % (D * 16);
    const int r = 8 * rg + ((lane & 31) >> 2);
    const int c = 4 * (in / 512) + ((lane & 3) ^ ((r >> 2) & 3));
    const u16* p = src + row_of(x0 + r) * stride + c * 8;
    __builtin_amdgcn_global_load_lds((gbl_void*)p, (lds_void*)(dst + piece * 1024), 16, 0, 0);
  }
}

// Tile image: 8-row x 32-column subtiles of 512 B with the chunks of a row rotated by its row
// group: conflict-free for row reads and for transposed reads. DK, DV: multiples of 32.
template <int DK, int DV>
__global__ void __launch_bounds__(512) swa_prefill32_kernel(SwaArgs a) {
  constexpr int KC = DK / 16, DBK = DV / 32;
  constexpr int RGK = DK * 16, RGV = DV * 16;                  // bytes of an 8-row group
  constexpr int TILE_K = KT * DK * 2, TILE_B = KT * (DK + DV) * 2, NBUF = 3;
  constexpr int NPK = DK / 8, NPV = DV / 8;                    // 1-KiB pieces of a tile
  extern __shared__ __attribute__((aligned(16))) char lds[];   // [NBUF][K tile | V tile], slot table
  int* table = (int*)(lds + NBUF * TILE_B);
  const int s = blockIdx.y, h = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wid = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int qc = lane & 31, hi = lane >> 5;
  const int t0 = a.cu[s], len = a.cu[s + 1] - t0;
  const int blk = (int)(gridDim.x - 1 - blockIdx.x);           // longest lists first
  const int wg_q0 = blk * LROWS;
  if (wg_q0 >= len) return;                                    // workgroup-uniform
  const int p0 = a.positions[t0];
  const int q0 = wg_q0 + wid * 32;
  const bool active = q0 < len;
  const int kvh = h / (a.H / a.G);
  const KeyList kl(p0 + wg_q0, p0 + min(wg_q0 + LROWS, len) - 1, a.window, a.keep);
  const int ntiles = (kl.n + KT - 1) / KT;
  const int* bt = a.block_tables + (long)s * a.bt_stride;
  const auto row_of = [&](int x) {
    const int j = kl.key(x);
    return bt[j / a.block_size] * a.block_size + j % a.block_size;
  };
  const bool use_table = kl.n <= a.table_cap;
  if (use_table)
    for (int x = tid; x < kl.n; x += 512) table[x] = row_of(x);

  bf16x8 qf[KC];
  {
    const u16* qp = a.q + (long)(t0 + min(q0 + qc, len - 1)) * a.ldq + (long)h * DK + 8 * hi;
#pragma unroll
    for (int c = 0; c < KC; ++c) {
      const uint4 v = *reinterpret_cast<const uint4*>(qp + 16 * c);
      qf[c] = *reinterpret_cast<const bf16x8*>(&v);
    }
  }
  const int qpos = p0 + q0 + qc;
  const int wq_lo = p0 + q0, wq_hi = p0 + min(q0 + 32, len) - 1;
  f32x16 o[DBK];
#pragma unroll
  for (int i = 0; i < DBK; ++i)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[i][r] = 0.f;
  float m_run = -INFINITY, l_part = 0.f;
  __syncthreads();

  const auto row_in_list = [&](int x) -> long {
    x = min(x, kl.n - 1);
    return use_table ? table[x] : row_of(x);
  };
  const auto stage = [&](int buf, int x0) {
    char* kd = lds + buf * TILE_B;
    stage_rows<DK>(a.k + kvh * DK, a.k_stride, kd, x0, wid, lane, row_in_list);
    stage_rows<DV>(a.v + kvh * DV, a.v_stride, kd + TILE_K, x0, wid, lane, row_in_list);
  };
  const auto wait_one_tile = [&]() {                           // all but the youngest tile landed
    constexpr int LO = NPK / 8 + NPV / 8, RK = NPK % 8, RV = NPV % 8;
    static_assert(LO + 2 < 16, "vmcnt field");
    const int extra = (wid < RK) + (wid < RV);                 // wave-uniform
    constexpr int BASE = (7 << 4) | (15 << 8);                 // other counters at their maxima
    if (extra == 0) __builtin_amdgcn_s_waitcnt(LO | BASE);
    else if (extra == 1) __builtin_amdgcn_s_waitcnt((LO + 1) | BASE);
    else __builtin_amdgcn_s_waitcnt((LO + 2) | BASE);
    asm volatile("" ::: "memory");
  };
  stage(0, 0);
  if (ntiles > 1) {
    stage(1, KT);
    wait_one_tile();
  } else {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  }
  __syncthreads();
  const int g16 = lane >> 4, q4 = (lane >> 2) & 3, p4 = lane & 3;
  int kbase[2], vbase[2];
#pragma unroll
  for (int par = 0; par < 2; ++par)
    kbase[par] = RGK * (qc >> 3) + 64 * (qc & 7) + 16 * ((2 * par + hi) ^ ((qc >> 2) & 3));
  {
    const int cl = 2 * (g16 & 1) + (p4 >> 1);
    vbase[0] = 64 * (4 * hi + q4) + 16 * (cl ^ hi) + 8 * (p4 & 1);
    vbase[1] = RGV + 64 * (4 * hi + q4) + 16 * (cl ^ (hi ^ 2)) + 8 * (p4 & 1);
  }
  f32x16 sacc[2];
  int cur = 0;
  for (int t = 0; t < ntiles; ++t) {
    const int x0 = t * KT;
    if (t + 2 < ntiles) stage(cur == 0 ? 2 : cur - 1, x0 + 2 * KT);
    const int kt0 = kl.key(x0), kt1 = kl.key(x0 + KT - 1);     // the tile's first and last key
    // tiles above this wave's rows, or all of them past its window and not kept, are skipped
    if (active && kt0 <= wq_hi && (kt1 > wq_lo - a.window || kt0 < a.keep)) {
      const char* kt = lds + cur * TILE_B;
#pragma unroll
      for (int sub = 0; sub < 2; ++sub) {
#pragma unroll
        for (int r = 0; r < 16; ++r) sacc[sub][r] = 0.f;
#pragma unroll
        for (int c = 0; c < KC; ++c) {
          const bf16x8 kf = *reinterpret_cast<const bf16x8*>(
              kt + kbase[c & 1] + 4 * RGK * sub + 512 * (c >> 1));
          sacc[sub] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[c], sacc[sub], 0, 0, 0);
        }
      }
      // only tiles that cross this wave's diagonal or the window's far edge are masked
      if (kt1 > wq_lo || wq_hi - kt0 >= a.window) {
#pragma unroll
        for (int sub = 0; sub < 2; ++sub)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int key = kl.key(x0 + 32 * sub + (r & 3) + 8 * (r >> 2) + 4 * hi);
            if (key > qpos || (qpos - key >= a.window && key >= a.keep)) sacc[sub][r] = -INFINITY;
          }
      }
      float mloc = max3(sacc[0][0], sacc[0][1], sacc[0][2]);
#pragma unroll
      for (int r = 3; r < 15; r += 2) mloc = max3(mloc, sacc[0][r], sacc[0][r + 1]);
      mloc = max3(mloc, sacc[0][15], sacc[1][0]);
#pragma unroll
      for (int r = 1; r < 15; r += 2) mloc = max3(mloc, sacc[1][r], sacc[1][r + 1]);
      mloc = fmaxf(mloc, sacc[1][15]);
      mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
      float alpha = 1.f;
      if ((mloc - m_run) * a.scale_log2 > RESCALE_THR) {
        alpha = m_run == -INFINITY ? 0.f
                                   : __builtin_amdgcn_exp2f((m_run - mloc) * a.scale_log2);
        m_run = mloc;
      }
      const float mc = (m_run == -INFINITY ? 0.f : m_run) * a.scale_log2;
      float psum = 0.f;
#pragma unroll
      for (int sub = 0; sub < 2; ++sub)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const float e = __builtin_amdgcn_exp2f(fmaf(sacc[sub][r], a.scale_log2, -mc));
          sacc[sub][r] = e;
          psum += e;
        }
      l_part = l_part * alpha + psum;
      if (__ballot(alpha != 1.f)) {
#pragma unroll
        for (int i = 0; i < DBK; ++i)
#pragma unroll
          for (int r = 0; r < 16; ++r) o[i][r] *= alpha;
      }
      const char* vt = kt + TILE_K;
#pragma unroll
      for (int ks = 0; ks < 4; ++ks) {
        const int sub = ks >> 1, hs = ks & 1;
        bf16x8 pb;
#pragma unroll
        for (int j = 0; j < 8; ++j) pb[j] = (__bf16)sacc[sub][8 * hs + j];
#pragma unroll
        for (int db = 0; db < DBK; ++db) {
          const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
              (__attribute__((address_space(3))) s16x4*)(vt + vbase[0] + 2 * RGV * ks + 512 * db));
          const s16x4 up = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
              (__attribute__((address_space(3))) s16x4*)(vt + vbase[1] + 2 * RGV * ks + 512 * db));
          const s16x8 w = {lo[0], lo[1], lo[2], lo[3], up[0], up[1], up[2], up[3]};
          o[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8*>(&w),
                                                         pb, o[db], 0, 0, 0);
        }
      }
    }
    if (t + 2 < ntiles) wait_one_tile();
    else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_waitcnt(0xC07F);                          // lgkmcnt(0): own reads done
    __builtin_amdgcn_s_barrier();
    cur = (cur == 2) ? 0 : cur + 1;
  }
  if (!active) return;
  const float l_tot = l_part + __shfl_xor(l_part, 32, 64);
  const float inv = l_tot > 0.f ? 1.f / l_tot : 0.f;
  const int qr = q0 + qc;
  if (qr < len) {
    u16* op = a.out + (long)(t0 + qr) * a.ldo + (long)h * DV;
    const float* gp = a.gate ? a.gate + (long)(t0 + qr) * a.ldg + (long)h * DV : nullptr;
#pragma unroll
    for (int db = 0; db < DBK; ++db)
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        f32x4 w = {1.f, 1.f, 1.f, 1.f};
        if (gp != nullptr) {
          w = *reinterpret_cast<const f32x4*>(gp + 32 * db + 8 * g + 4 * hi);
#pragma unroll
          for (int r = 0; r < 4; ++r) w[r] = sigmoid32(w[r]);
        }
        U16x4 v;
#pragma unroll
        for (int r = 0; r < 4; ++r) v.v[r] = f2bf(o[db][4 * g + r] * inv * w[r]);
        *reinterpret_cast<U16x4*>(op + 32 * db + 8 * g + 4 * hi) = v;
      }
  }
}

// 4 waves x 16 query rows of one head
template <int DK, int DV>
__global__ void __launch_bounds__(256) swa_prefill16_kernel(SwaArgs a) {
  constexpr int KK = DK / 32, DB = DV / 16, ROWK = DK + 16, ROWV = DV + 16;
  constexpr int CHK = DK / 8, CHV = DV / 8, PK = KT * CHK / 256, PV = KT * CHV / 256;
  __shared__ __attribute__((aligned(16))) u16 ktile[KT * ROWK];
  __shared__ __attribute__((aligned(16))) u16 vtile[KT * ROWV];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int s = blockIdx.y, h = blockIdx.z;
  const int col = lane & 15, grp = lane >> 4;
  const int t0 = a.cu[s], len = a.cu[s + 1] - t0;
  const int wg_q0 = blockIdx.x * 64;
  if (wg_q0 >= len) return;                                      // workgroup-uniform
  const int p0 = a.positions[t0];
  const int q0 = wg_q0 + wid * 16;
  const bool active = q0 < len;
  const int kvh = h / (a.H / a.G);
  const KeyList kl(p0 + wg_q0, p0 + min(wg_q0 + 64, len) - 1, a.window, a.keep);
  const int* bt = a.block_tables + (long)s * a.bt_stride;
  bf16x8 qf[KK];
  {
    const u16* qp = a.q + (long)(t0 + min(q0 + col, len - 1)) * a.ldq + (long)h * DK;
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) {
      const uint4 v = *reinterpret_cast<const uint4*>(qp + kk * 32 + grp * 8);
      qf[kk] = *reinterpret_cast<const bf16x8*>(&v);
    }
  }
  const int my_q = p0 + q0 + col, wq_lo = p0 + q0, wq_hi = p0 + min(q0 + 16, len) - 1;
  float m_run = -INFINITY, l_part = 0.f;
  f32x4 o_acc[DB];
#pragma unroll
  for (int i = 0; i < DB; ++i) o_acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  // the next tile in flight in registers (of a native vector type: arrays of
  // HIP's uint4 would be kept in memory)
  u32x4 kr[PK], vr[PV];
  const auto row_at = [&](int x) {
    const int key = kl.key(min(x, kl.n - 1));
    return (long)bt[key / a.block_size] * a.block_size + key % a.block_size;
  };
  const auto load_tile = [&](int x0) {
#pragma unroll
    for (int j = 0; j < PK; ++j) {
      const int i = tid + 256 * j;
      kr[j] = *reinterpret_cast<const u32x4*>(a.k + row_at(x0 + i / CHK) * a.k_stride + kvh * DK +
                                              (i % CHK) * 8);
    }
#pragma unroll
    for (int j = 0; j < PV; ++j) {
      const int i = tid + 256 * j;
      vr[j] = *reinterpret_cast<const u32x4*>(a.v + row_at(x0 + i / CHV) * a.v_stride + kvh * DV +
                                              (i % CHV) * 8);
    }
  };
  load_tile(0);
  const int qrow = (lane >> 2) & 3, pcol = lane & 3;
  for (int x0 = 0; x0 < kl.n; x0 += KT) {
    __syncthreads();                                             // previous tile fully read
#pragma unroll
    for (int j = 0; j < PK; ++j) {
      const int i = tid + 256 * j;
      *reinterpret_cast<u32x4*>(ktile + i / CHK * ROWK + i % CHK * 8) = kr[j];
    }
#pragma unroll
    for (int j = 0; j < PV; ++j) {
      const int i = tid + 256 * j;
      *reinterpret_cast<u32x4*>(vtile + i / CHV * ROWV + i % CHV * 8) = vr[j];
    }
    __syncthreads();
    if (x0 + KT < kl.n) load_tile(x0 + KT);                      // in flight during compute
    const int kt0 = kl.key(x0), kt1 = kl.key(x0 + KT - 1);
    if (!active || kt0 > wq_hi || (kt1 <= wq_lo - a.window && kt0 >= a.keep)) continue;
    f32x4 s_acc[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const u16* kp = ktile + (16 * u + col) * ROWK;
      s_acc[u] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < KK; ++kk)
        s_acc[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            *reinterpret_cast<const bf16x8*>(kp + kk * 32 + grp * 8), qf[kk], s_acc[u], 0, 0, 0);
    }
    float p[16], tmax = -INFINITY;
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = kl.key(x0 + 16 * u + 4 * grp + r);
        const bool seen = key <= my_q && (my_q - key < a.window || key < a.keep);
        const float v = seen ? s_acc[u][r] * a.scale_log2 : -INFINITY;
        p[u * 4 + r] = v;
        tmax = fmaxf(tmax, v);
      }
    tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
    const float m_new = fmaxf(m_run, tmax);
    const float m_use = m_new == -INFINITY ? 0.f : m_new;        // nothing seen yet: keep it finite
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_use);
    m_run = m_new;
    float psum = 0.f;
#pragma unroll
    for (int j = 0; j < 16; ++j) { p[j] = __builtin_amdgcn_exp2f(p[j] - m_use); psum += p[j]; }
    l_part = l_part * alpha + psum;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float al = __shfl(alpha, 4 * grp + r, 64);
#pragma unroll
      for (int i = 0; i < DB; ++i) o_acc[i][r] *= al;
    }
    // O += P . V, two 32-key halves; B operand rows: keys 32 hh + 4 grp + q and 16 further on
#pragma unroll
    for (int hh = 0; hh < 2; ++hh) {
      bf16x8 pa;
#pragma unroll
      for (int j = 0; j < 8; ++j) pa[j] = (__bf16)p[8 * hh + j];
#pragma unroll
      for (int i = 0; i < DB; ++i) {
        const u16* a0 = vtile + (32 * hh + 4 * grp + qrow) * ROWV + 16 * i + 4 * pcol;
        const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (__attribute__((address_space(3))) s16x4*)(a0));
        const s16x4 up = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (__attribute__((address_space(3))) s16x4*)(a0 + 16 * ROWV));
        const s16x8 w = {lo[0], lo[1], lo[2], lo[3], up[0], up[1], up[2], up[3]};
        o_acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            pa, *reinterpret_cast<const bf16x8*>(&w), o_acc[i], 0, 0, 0);
      }
    }
  }
  if (!active) return;
  float l_tot = l_part + __shfl_xor(l_part, 16, 64);
  l_tot += __shfl_xor(l_tot, 32, 64);
  const float inv = l_tot > 0.f ? 1.f / l_tot : 0.f;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const float iv = __shfl(inv, 4 * grp + r, 64);
    const int qr = q0 + 4 * grp + r;
    if (qr < len) {
      u16* op = a.out + (long)(t0 + qr) * a.ldo + (long)h * DV;
      const float* gp = a.gate ? a.gate + (long)(t0 + qr) * a.ldg + (long)h * DV : nullptr;
#pragma unroll
      for (int i = 0; i < DB; ++i) {
        float v = o_acc[i][r] * iv;
        if (gp != nullptr) v *= sigmoid32(gp[16 * i + col]);
        op[16 * i + col] = f2bf(v);
      }
    }
  }
}

// One query token a sequence. Workgroup = 4 waves of one (sequence, kv head, chunk of HP heads,
// key split); a wave takes every fourth 32-key tile of the split.
template <int DK, int DV, int HP>
__global__ void __launch_bounds__(256) swa_decode_kernel(SwaArgs a) {
  constexpr int KK = DK / 32, LPR = DV / 8;        // lanes that cover a V row with 16 bytes each
  constexpr int KPI = 64 / LPR, NV = 32 / KPI;     // keys per V load of a wave, V loads per tile
  static_assert(32 % KPI == 0, "V loads tile 32 keys");
  __shared__ __attribute__((aligned(16))) float pl[4][32][HP];
  __shared__ __attribute__((aligned(16))) float ol[4][HP][DV];
  __shared__ float ml[4][HP][2];
  const int rep = a.H / a.G, nhc = (rep + HP - 1) / HP;
  const int s = blockIdx.y, split = blockIdx.z;
  const int kvh = blockIdx.x / nhc, h0 = kvh * rep + (blockIdx.x % nhc) * HP;
  const int nh = min(HP, (kvh + 1) * rep - h0);
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int fr = lane & 15, fq = lane >> 4;
  const int t = a.cu[s];
  if (a.cu[s + 1] <= t) return;
  const int p = a.positions[t];
  const KeyList kl(p, p, a.window, a.keep);
  const int* bt = a.block_tables + (long)s * a.bt_stride;
  const int ntiles = (kl.n + 31) / 32, per = (ntiles + a.nsplit - 1) / a.nsplit;
  const int tile_hi = min(ntiles, (split + 1) * per);
  bf16x8 qf[KK];
#pragma unroll
  for (int kk = 0; kk < KK; ++kk) {
    uint4 v = uint4{0u, 0u, 0u, 0u};
    if (fr < nh)
      v = *reinterpret_cast<const uint4*>(a.q + (long)t * a.ldq + (long)(h0 + fr) * DK + kk * 32 +
                                          fq * 8);
    qf[kk] = *reinterpret_cast<const bf16x8*>(&v);
  }
  float m_run = -INFINITY, l_run = 0.f;            // of head fr
  float acc[HP][8];
#pragma unroll
  for (int h = 0; h < HP; ++h)
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[h][i] = 0.f;
  for (int tile = split * per + wid; tile < tile_hi; tile += 4) {
    const int x0 = tile * 32;
    const int key = kl.key(min(x0 + (lane & 31), kl.n - 1));
    const int row = bt[key / a.block_size] * a.block_size + key % a.block_size;
    bf16x8 kf[2][KK];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const long r = __shfl(row, 16 * u + fr, 64);
#pragma unroll
      for (int kk = 0; kk < KK; ++kk) {
        const uint4 v = *reinterpret_cast<const uint4*>(a.k + r * a.k_stride + kvh * DK + kk * 32 +
                                                        fq * 8);
        kf[u][kk] = *reinterpret_cast<const bf16x8*>(&v);
      }
    }
    uint4 vv[NV];
    // (widths whose rows do not tile a wave leave its last lanes to repeat the last key's row)
    const int vk = min(lane / LPR, KPI - 1);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const long r = __shfl(row, i * KPI + vk, 64);
      vv[i] = *reinterpret_cast<const uint4*>(a.v + r * a.v_stride + kvh * DV + (lane % LPR) * 8);
    }
    f32x4 sa[2];
    float tmax = -INFINITY;
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      sa[u] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < KK; ++kk)
        sa[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[u][kk], qf[kk], sa[u], 0, 0, 0);
      // lane: head fr, keys x0 + 16 u + 4 fq + r; every listed key is seen
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        sa[u][r] = x0 + 16 * u + 4 * fq + r < kl.n ? sa[u][r] * a.scale_log2 : -INFINITY;
        tmax = fmaxf(tmax, sa[u][r]);
      }
    }
    tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
    const float m_new = fmaxf(m_run, tmax);        // finite: a tile holds at least one key
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
    m_run = m_new;
    float psum = 0.f;
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float e = __builtin_amdgcn_exp2f(sa[u][r] - m_new);
        psum += e;
        if (fr < HP) pl[wid][16 * u + 4 * fq + r][fr] = e;
      }
    l_run = l_run * alpha + psum;                  // this lane's keys only
    if (__ballot(fr < nh && alpha != 1.f)) {
#pragma unroll
      for (int h = 0; h < HP; ++h) {
        const float al = __shfl(alpha, h, 64);
#pragma unroll
        for (int i = 0; i < 8; ++i) acc[h][i] *= al;
      }
    }
    // the wave's own weights, written above by its own lanes: in order in the LDS pipe
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      float v8[8];
      unpack8bf(vv[i], v8);
      const float* pr = pl[wid][i * KPI + vk];
#pragma unroll
      for (int h = 0; h < HP; ++h) {
        const float w = pr[h];
#pragma unroll
        for (int c = 0; c < 8; ++c) acc[h][c] += w * v8[c];
      }
    }
    __builtin_amdgcn_wave_barrier();
  }
  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  if (lane < HP) { ml[wid][lane][0] = m_run; ml[wid][lane][1] = l_run; }
#pragma unroll
  for (int h = 0; h < HP; ++h)
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      float v = acc[h][i];
      if constexpr ((LPR & (LPR - 1)) == 0) {
#pragma unroll
        for (int o = LPR; o < 64; o <<= 1) v += __shfl_xor(v, o, 64);
      } else {                                     // lanes below LPR gather their column's sums
        const float own = v;
#pragma unroll
        for (int k = 1; k < KPI; ++k) v += __shfl(own, (lane + k * LPR) & 63, 64);
      }
      acc[h][i] = v;
    }
  if (lane < LPR) {
#pragma unroll
    for (int h = 0; h < HP; ++h) {
      *reinterpret_cast<f32x4*>(&ol[wid][h][lane * 8]) =
          f32x4{acc[h][0], acc[h][1], acc[h][2], acc[h][3]};
      *reinterpret_cast<f32x4*>(&ol[wid][h][lane * 8 + 4]) =
          f32x4{acc[h][4], acc[h][5], acc[h][6], acc[h][7]};
    }
  }
  __syncthreads();
  const int S = gridDim.y;
  float* stats = a.ws;
  float* part = a.ws + stat_floats(a.nsplit, S, a.H);
  for (int i = tid; i < nh * DV; i += 256) {
    const int h = i / DV, c = i % DV;
    float M = -INFINITY;
#pragma unroll
    for (int w = 0; w < 4; ++w) M = fmaxf(M, ml[w][h][0]);
    float L = 0.f, o = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      if (ml[w][h][0] == -INFINITY) continue;      // a wave without tiles
      const float e = __builtin_amdgcn_exp2f(ml[w][h][0] - M);
      L += ml[w][h][1] * e;
      o += ol[w][h][c] * e;
    }
    if (a.nsplit == 1) {
      const int oc = (h0 + h) * DV + c;
      float v = o / L;
      if (a.gate != nullptr) v *= sigmoid32(a.gate[(long)t * a.ldg + oc]);
      a.out[(long)t * a.ldo + oc] = f2bf(v);
    } else {
      const long b = ((long)split * S + s) * a.H + h0 + h;
      part[b * DV + c] = o;
      if (c == 0) { stats[2 * b] = M; stats[2 * b + 1] = L; }
    }
  }
}

// out = the splits' un-normalised partial sums, weighed by their (max, sum); 4 columns a thread
template <int DV>
__global__ void __launch_bounds__(256) swa_reduce_kernel(SwaArgs a, int S) {
  const long gid = (long)blockIdx.x * blockDim.x + threadIdx.x;
  const int w4 = a.H * DV / 4;
  if (gid >= (long)S * w4) return;
  const int s = (int)(gid / w4), c = (int)(gid % w4) * 4, h = c / DV;
  if (a.cu[s + 1] <= a.cu[s]) return;
  const float* stats = a.ws;
  const float* part = a.ws + stat_floats(a.nsplit, S, a.H);
  float M = -INFINITY;
  for (int k = 0; k < a.nsplit; ++k) M = fmaxf(M, stats[2 * (((long)k * S + s) * a.H + h)]);
  float L = 0.f;
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
  for (int k = 0; k < a.nsplit; ++k) {
    const long b = ((long)k * S + s) * a.H + h;
    if (stats[2 * b] == -INFINITY) continue;       // a split without keys
    const float e = __builtin_amdgcn_exp2f(stats[2 * b] - M);
    L += stats[2 * b + 1] * e;
    o += e * *reinterpret_cast<const f32x4*>(part + b * DV + c % DV);
  }
  o *= 1.f / L;
  if (a.gate != nullptr) {
    const f32x4 g = *reinterpret_cast<const f32x4*>(a.gate + (long)a.cu[s] * a.ldg + c);
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] *= sigmoid32(g[i]);
  }
  uint2 pk;
  pk.x = pack2bf(o[0], o[1]);
  pk.y = pack2bf(o[2], o[3]);
  *reinterpret_cast<uint2*>(a.out + (long)a.cu[s] * a.ldo + c) = pk;
}

int decode_splits(int num_seqs, int H, int G, long keys) {
  const int rep = H / G, hp = rep <= 4 ? 4 : 8;
  const long base = (long)num_seqs * G * ((rep + hp - 1) / hp);
  long n = (1536 + base - 1) / base;
  const long most = (keys + 127) / 128;            // a tile for each wave of a workgroup
  n = n > most ? most : n;
  n = n > 32 ? 32 : n;
  return n < 1 ? 1 : (int)n;
}

// key / value widths this file is built for
#define SWA_WIDTHS(F) F(64, 64) F(128, 128) F(64, 128) F(96, 192) F(128, 256)

template <int DK, int DV>
int launch_swa(SwaArgs a, int num_seqs, int max_seqlen, hipStream_t st) {
  if (max_seqlen == 1) {
    const int rep = a.H / a.G, hp = rep <= 4 ? 4 : 8;
    dim3 grid(a.G * ((rep + hp - 1) / hp), num_seqs, a.nsplit);
    if (hp == 4) swa_decode_kernel<DK, DV, 4><<<grid, 256, 0, st>>>(a);
    else swa_decode_kernel<DK, DV, 8><<<grid, 256, 0, st>>>(a);
    if (a.nsplit > 1) {
      const long n = (long)num_seqs * a.H * DV / 4;
      swa_reduce_kernel<DV><<<(int)((n + 255) / 256), 256, 0, st>>>(a, num_seqs);
    }
    DLI_RETURN_LAUNCH();
  }
  if (max_seqlen < 192) {
    dim3 grid((max_seqlen + 63) / 64, num_seqs, a.H);
    swa_prefill16_kernel<DK, DV><<<grid, 256, 0, st>>>(a);
    DLI_RETURN_LAUNCH();
  }
  const long list = (long)a.window + LROWS + a.keep;
  constexpr int TILES = 3 * KT * (DK + DV) * 2;
  a.table_cap = list <= 6144 && TILES + list * 4 + 16 <= 160 * 1024 ? (int)list : 0;
  const int sh = TILES + a.table_cap * 4 + 16;
  static bool raised = false;
  if (!raised) {
    const hipError_t e = hipFuncSetAttribute((const void*)swa_prefill32_kernel<DK, DV>,
                                             hipFuncAttributeMaxDynamicSharedMemorySize,
                                             160 * 1024);
    if (e != hipSuccess) return (int)e;
    raised = true;
  }
  dim3 grid((max_seqlen + LROWS - 1) / LROWS, num_seqs, a.H);
  swa_prefill32_kernel<DK, DV><<<grid, 512, sh, st>>>(a);
  DLI_RETURN_LAUNCH();
}

}  // namespace

// Workspace bytes of a decode step (0: not split over keys)
extern "C" long dli_swa_attention_workspace_bytes(int num_seqs, int max_seqlen, int H, int G,
                                                  int dv, int window, int keep) {
  if (max_seqlen != 1 || H < 1 || G < 1) return 0;
  const int n = decode_splits(num_seqs, H, G, (long)window + keep);
  return n == 1 ? 0 : (stat_floats(n, num_seqs, H) + (long)n * num_seqs * H * dv) * 4;
}

// Returns hipErrorNotSupported (801) for shapes this family does not take. A decode step
// (max_seqlen 1) gets the workspace its query asked for.
extern "C" int dli_swa_attention(const void* q, int ldq, const void* k, long k_stride,
                                 const void* v, long v_stride, void* out, int ldo, const int* cu,
                                 const int* positions, const int* block_tables, int bt_stride,
                                 int block_size, int num_seqs, int max_seqlen, int H, int G,
                                 int dk, int dv, int window, int keep, float scale,
                                 const float* gate, int ldg, void* ws, hipStream_t st) {
  if (num_seqs <= 0 || max_seqlen <= 0) return 0;
  if (H < 1 || G < 1 || H % G || window < 1 || keep < 0 || block_size < 1)
    return (int)hipErrorInvalidValue;
  const bool aligned = (((uintptr_t)q | (uintptr_t)k | (uintptr_t)v) & 15) == 0 &&
                       (uintptr_t)out % 8 == 0 && ldq % 8 == 0 && k_stride % 8 == 0 &&
                       v_stride % 8 == 0 && ldo % 4 == 0 &&
                       (gate == nullptr || ((uintptr_t)gate % 16 == 0 && ldg % 4 == 0));
  if (!aligned || !(scale > 0.f) || num_seqs > 65535 || H > 65535)
    return (int)hipErrorNotSupported;
  SwaArgs a{(const u16*)q, ldq, (const u16*)k, k_stride, (const u16*)v, v_stride, (u16*)out, ldo,
            gate, ldg, cu, positions, block_tables, bt_stride, block_size, H, G, window, keep,
            scale * LOG2E, 0, 1, (float*)ws};
  if (max_seqlen == 1) {
    a.nsplit = decode_splits(num_seqs, H, G, (long)window + keep);
    if (a.nsplit > 1 && ws == nullptr) return (int)hipErrorInvalidValue;
  }
#define SWA_TRY(K, V) if (dk == K && dv == V) return launch_swa<K, V>(a, num_seqs, max_seqlen, st);
  SWA_WIDTHS(SWA_TRY)
#undef SWA_TRY
  return (int)hipErrorNotSupported;
}
