// Rotated queries and keys of the hybrid family (models/mixers.py, ops/hybrid.py). S = storage
// type (u16 = bf16 bits, or float); projections, tables and arithmetic are fp32.
//
//  * rotation_table  cosines | sines of position * freq for every token of a step, made once
//                    per step and rotation: the angle is formed in double and rounded once
//  * rope_prepare    q / k (/ v) of an attention with rotated queries and keys: bias, the
//                    rotation of the first `rot` dims of every head (dimension i with i +
//                    rot/2, or 2i with 2i + 1), rotated k and v -> cache rows, q -> S. tied: there
//                    is no v, the value row is the key before its rotation. G = 0: queries only.
#include "common.h"

namespace {

template <typename S> __device__ __forceinline__ float ldf(const S* p);
template <> __device__ __forceinline__ float ldf<u16>(const u16* p) { return bf2f(*p); }
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <typename S> __device__ __forceinline__ void stf(S* p, float v);
template <> __device__ __forceinline__ void stf<u16>(u16* p, float v) { *p = f2bf(v); }
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }

__global__ void __launch_bounds__(256) rotation_table_kernel(
    float* __restrict__ out, const int* __restrict__ positions, const double* __restrict__ freq,
    int T, int n) {
  const long gid = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (gid >= (long)T * n) return;
  const int t = (int)(gid / n), i = (int)(gid % n);
  const double a = (double)positions[t] * freq[i];
  out[(long)t * 2 * n + i] = (float)cos(a);
  out[(long)t * 2 * n + n + i] = (float)sin(a);
}

// VEC consecutive elements (aligned: VEC = 4 takes 16-byte fp32 / 8-byte bf16 accesses)
template <int VEC> __device__ __forceinline__ void ldv(const float* p, float* v) {
  if constexpr (VEC == 4) {
    const f32x4 q = *reinterpret_cast<const f32x4*>(p);
    v[0] = q[0]; v[1] = q[1]; v[2] = q[2]; v[3] = q[3];
  } else {
    v[0] = *p;
  }
}
template <typename S, int VEC> __device__ __forceinline__ void stv(S* p, const float* v) {
  if constexpr (VEC == 4 && sizeof(S) == 2) {
    uint2 pk;
    pk.x = pack2bf(v[0], v[1]);
    pk.y = pack2bf(v[2], v[3]);
    *reinterpret_cast<uint2*>(p) = pk;
  } else if constexpr (VEC == 4) {
    *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
  } else {
    stf(p, v[0]);
  }
}

// One thread per unit: VEC rotated pairs (two column groups), or VEC columns that pass.
// Units of a token: H + G heads of up = (rot/2 + d - rot) / VEC units, then G*dv/VEC value
// units (none when tied).
template <typename S, int VEC>
__global__ void __launch_bounds__(256) rope_prepare_kernel(
    const float* __restrict__ proj, int ldp, const S* __restrict__ bias,
    const float* __restrict__ table, int rot, int T, int H, int G, int d, int dv, int tied,
    S* __restrict__ q_out, S* __restrict__ kcache, S* __restrict__ vcache,
    const int* __restrict__ slots) {
  const int hr = rot >> 1;
  const int rp = hr / VEC, up = rp + (d - rot) / VEC;
  const int nu = (H + G) * up + (tied ? 0 : G * dv / VEC);
  const long gid = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (gid >= (long)T * nu) return;
  const int t = (int)(gid / nu), u = (int)(gid - (long)t * nu);
  const float* row = proj + (long)t * ldp;
  if (u >= (H + G) * up) {                           // a value group
    const int slot = slots[t];
    if (slot < 0) return;
    const int c = (u - (H + G) * up) * VEC, src = (H + G) * d + c;
    float v[VEC];
    ldv<VEC>(row + src, v);
    if (bias != nullptr) {
#pragma unroll
      for (int i = 0; i < VEC; ++i) v[i] += ldf(bias + src + i);
    }
    stv<S, VEC>(vcache + (long)slot * G * dv + c, v);
    return;
  }
  const int h = u / up, k = u - h * up;
  const bool pair = k < rp;
  const int c = pair ? k * VEC : rot + (k - rp) * VEC;
  const bool is_q = h < H;
  const int slot = is_q ? 0 : slots[t];
  if (slot < 0) return;
  const int src = h * d + c;
  float a[VEC], b[VEC];
  ldv<VEC>(row + src, a);
  if (pair) ldv<VEC>(row + src + hr, b);
  if (bias != nullptr) {
#pragma unroll
    for (int i = 0; i < VEC; ++i) {
      a[i] += ldf(bias + src + i);
      if (pair) b[i] += ldf(bias + src + hr + i);
    }
  }
  S* dst = is_q ? q_out + (long)t * H * d + src : kcache + (long)slot * G * d + (src - H * d);
  if (!is_q && tied && vcache != kcache) {           // tied values: the key before its rotation
    S* vd = vcache + (long)slot * G * d + (src - H * d);
    stv<S, VEC>(vd, a);
    if (pair) stv<S, VEC>(vd + hr, b);
  }
  if (pair) {
    float cs[VEC], sn[VEC], x[VEC], y[VEC];
    ldv<VEC>(table + (long)t * rot + c, cs);
    ldv<VEC>(table + (long)t * rot + hr + c, sn);
#pragma unroll
    for (int i = 0; i < VEC; ++i) {
      x[i] = a[i] * cs[i] - b[i] * sn[i];
      y[i] = b[i] * cs[i] + a[i] * sn[i];
    }
    stv<S, VEC>(dst, x);
    stv<S, VEC>(dst + hr, y);
  } else {
    stv<S, VEC>(dst, a);
  }
}

// The same for adjacent pairs (2i, 2i + 1). A unit is 2 VEC columns of a rotated part (VEC pairs), or
// 2 VEC columns that pass (the last unit of a head may be cut short: VEC = 1, odd widths).
template <typename S, int VEC>
__global__ void __launch_bounds__(256) rope_prepare_adjacent_kernel(
    const float* __restrict__ proj, int ldp, const S* __restrict__ bias,
    const float* __restrict__ table, int rot, int T, int H, int G, int d, int dv, int tied,
    S* __restrict__ q_out, S* __restrict__ kcache, S* __restrict__ vcache,
    const int* __restrict__ slots) {
  constexpr int W = 2 * VEC;
  const int up = (d + W - 1) / W, uv = (dv + W - 1) / W;
  const int nu = (H + G) * up + (tied ? 0 : G * uv);
  const long gid = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (gid >= (long)T * nu) return;
  const int t = (int)(gid / nu), u = (int)(gid - (long)t * nu);
  const bool is_v = u >= (H + G) * up;
  const int uu = is_v ? u - (H + G) * up : u, per = is_v ? uv : up, width = is_v ? dv : d;
  const int h = uu / per, c = (uu - h * per) * W;
  const bool is_q = !is_v && h < H;
  const int slot = is_q ? 0 : slots[t];
  if (slot < 0) return;
  const int src = (is_v ? (H + G) * d : 0) + h * width + c;
  const float* row = proj + (long)t * ldp + src;
  const int n = min(W, width - c);
  float v[W];
  if constexpr (VEC == 2) {
    const f32x4 x = *reinterpret_cast<const f32x4*>(row);
    v[0] = x[0]; v[1] = x[1]; v[2] = x[2]; v[3] = x[3];
  } else {
    v[0] = row[0];
    v[1] = n > 1 ? row[1] : 0.f;
  }
  if (bias != nullptr) {
#pragma unroll
    for (int i = 0; i < W; ++i)
      if (i < n) v[i] += ldf(bias + src + i);
  }
  const auto put = [&](S* p) {
    if constexpr (VEC == 2) {
      if constexpr (sizeof(S) == 2) {
        uint2 pk;
        pk.x = pack2bf(v[0], v[1]);
        pk.y = pack2bf(v[2], v[3]);
        *reinterpret_cast<uint2*>(p) = pk;
      } else {
        *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
      }
    } else {
      stf(p, v[0]);
      if (n > 1) stf(p + 1, v[1]);
    }
  };
  if (is_v) {
    put(vcache + (long)slot * G * dv + h * dv + c);
    return;
  }
  if (!is_q && tied && vcache != kcache) put(vcache + (long)slot * G * d + (src - H * d));
  if (c < rot) {                                     // rot is even: whole pairs
#pragma unroll
    for (int i = 0; i < VEC; ++i) {
      const int k = (c >> 1) + i;
      if (2 * k >= rot) continue;
      const float cs = table[(long)t * rot + k], sn = table[(long)t * rot + (rot >> 1) + k];
      const float a = v[2 * i], b = v[2 * i + 1];
      v[2 * i] = a * cs - b * sn;
      v[2 * i + 1] = b * cs + a * sn;
    }
  }
  put(is_q ? q_out + (long)t * H * d + src : kcache + (long)slot * G * d + (src - H * d));
}

}  // namespace

extern "C" int dli_rotation_table(float* out, const int* positions, const double* freq, int T,
                                  int n, hipStream_t st) {
  if (T <= 0 || n <= 0) return 0;
  const long tot = (long)T * n;
  rotation_table_kernel<<<(int)((tot + 255) / 256), 256, 0, st>>>(out, positions, freq, T, n);
  DLI_RETURN_LAUNCH();
}

extern "C" int dli_rope_prepare(const float* proj, int ldp, const void* bias, const float* table,
                                int rot, int T, int H, int G, int d, int dv, int tied,
                                int adjacent, void* q_out, void* kcache, void* vcache, const int* slots, int dt,
                                hipStream_t st) {
  if (T <= 0) return 0;
  if (H < 1 || G < 0 || (G > 0 && (H % G || kcache == nullptr || vcache == nullptr)) || d < 1 || dv < 1 || rot < 0 || (rot & 1) || rot > d ||
      (rot > 0 && table == nullptr) || (tied && dv != d) || (dt != 0 && dt != 1))
    return (int)hipErrorInvalidValue;
  const uintptr_t mis = (uintptr_t)proj | (uintptr_t)table | (uintptr_t)q_out |
                        (uintptr_t)kcache | (uintptr_t)vcache;
  if (adjacent) {
    const bool v4 = d % 4 == 0 && dv % 4 == 0 && ldp % 4 == 0 && mis % 16 == 0;
    const int w = v4 ? 4 : 2;
    const long tot = (long)T * ((H + G) * ((d + w - 1) / w) + (tied ? 0 : G * ((dv + w - 1) / w)));
    const int blocks = (int)((tot + 255) / 256);
#define RA_LAUNCH(S, VV)                                                                        \
  rope_prepare_adjacent_kernel<S, VV><<<blocks, 256, 0, st>>>(                                  \
      proj, ldp, (const S*)bias, table, rot, T, H, G, d, dv, tied, (S*)q_out, (S*)kcache,       \
      (S*)vcache, slots)
    if (v4) { if (dt == 0) RA_LAUNCH(u16, 2); else RA_LAUNCH(float, 2); }
    else { if (dt == 0) RA_LAUNCH(u16, 1); else RA_LAUNCH(float, 1); }
#undef RA_LAUNCH
    DLI_RETURN_LAUNCH();
  }
  const bool v4 = d % 4 == 0 && dv % 4 == 0 && rot % 8 == 0 && ldp % 4 == 0 && mis % 16 == 0;
  const int V = v4 ? 4 : 1;
  const int up = (rot / 2 + d - rot) / V;
  const long tot = (long)T * ((H + G) * up + (tied ? 0 : G * dv / V));
  const int blocks = (int)((tot + 255) / 256);
#define RP_LAUNCH(S, VV)                                                                        \
  rope_prepare_kernel<S, VV><<<blocks, 256, 0, st>>>(proj, ldp, (const S*)bias, table, rot, T,  \
                                                     H, G, d, dv, tied, (S*)q_out, (S*)kcache,  \
                                                     (S*)vcache, slots)
  if (v4) { if (dt == 0) RP_LAUNCH(u16, 4); else RP_LAUNCH(float, 4); }
  else { if (dt == 0) RP_LAUNCH(u16, 1); else RP_LAUNCH(float, 1); }
#undef RP_LAUNCH
  DLI_RETURN_LAUNCH();
}
