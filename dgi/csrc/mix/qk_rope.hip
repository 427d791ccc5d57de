// dgi/csrc/mix/qk_rope.hip — rotary positions and the paged K/V write of attentions without a q / k norm.
//
// One workgroup per token reads its fused projection row [q: H*dk | k: G*dk | (v: G*dv) | ...] and
//   * replaces q by rot(q) in place,
//   * writes rot(k) into the key pages at the row's slot and, beside it, the row's values: the v columns, or with
//     `shared` the key columns themselves as projected (a mixer whose values are its unrotated keys has no v columns).
// rot() turns pairs of the first rd dims of every head by the row's position (cos_sin [max_pos, rd]: rd/2 cos | rd/2 sin,
// frequency scaling folded in): `half` pairs (i, i + rd/2), else (2i, 2i + 1); the other dims pass through.  fp32 math.
//
// Cache layout per layer: k [num_blocks, G, block_size, dk], v [num_blocks, G, block_size, dv].
#include "../common.h"

using namespace dgi;

namespace {

template <typename T> __device__ __forceinline__ float ldf(const T* p);
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldf<uint16_t>(const uint16_t* p) { return bf16_to_f32(*p); }
template <typename T> __device__ __forceinline__ void stf(T* p, float v);
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void stf<uint16_t>(uint16_t* p, float v) { *p = f32_to_bf16(v); }

// C elements as raw bits beside their floats: C = 1, or 16 bytes (8 bf16 / 4 fp32)
template <typename T, int C> struct Piece {
  float f[C];
  u32x4 raw;
  __device__ __forceinline__ void load(const T* p) {
    if constexpr (C == 1) {
      f[0] = ldf<T>(p);
    } else {
      raw = *reinterpret_cast<const u32x4*>(p);
      if constexpr (sizeof(T) == 2) unpack8(raw, f);
      else {
#pragma unroll
        for (int j = 0; j < 4; ++j) f[j] = __uint_as_float(raw[j]);
      }
    }
  }
  __device__ __forceinline__ void store_raw(T* p) const {
    if constexpr (C == 1) stf<T>(p, f[0]);           // a bf16 value survives the round trip bit for bit
    else *reinterpret_cast<u32x4*>(p) = raw;
  }
  static __device__ __forceinline__ void store(T* p, const float* v) {
    if constexpr (C == 1) stf<T>(p, v[0]);
    else if constexpr (sizeof(T) == 2) *reinterpret_cast<u32x4*>(p) = pack8(v);
    else *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  }
};

// C elements per piece.  HALF: a unit is the piece pair (e, e + rd/2); interleaved: C = 1: the pair (2u, 2u + 1),
// else a piece of C / 2 pairs.
template <typename T, int C, bool HALF>
__global__ __launch_bounds__(256) void qk_rope_kernel(T* __restrict__ qkv, int stride, const int* __restrict__ positions,
                                                      const int* __restrict__ slots, const float* __restrict__ cos_sin,
                                                      int rd, int H, int G, int dk, int dv, T* __restrict__ k_cache,
                                                      T* __restrict__ v_cache, int block_size, int shared) {
  using P = Piece<T, C>;
  constexpr bool PAIR = HALF || C == 1;              // two loads per rotated unit
  const int t = blockIdx.x;
  T* row = qkv + (size_t)t * stride;
  const int slot = slots[t];
  const int blk = slot >= 0 ? slot / block_size : 0;
  const int off = slot >= 0 ? slot - blk * block_size : 0;
  const int rh = rd >> 1;
  const float* cs = rd > 0 ? cos_sin + (size_t)positions[t] * rd : nullptr;
  const int nrot = PAIR ? rh / C : rd / C;           // rotated units per head
  const int npass = (dk - rd) / C;                   // pass-through units per key head
  const int nq = H * nrot;                           // q's other dims stay where they are
  const int total = nq + (slot >= 0 ? G * (nrot + npass) : 0);
  for (int i = threadIdx.x; i < total; i += 256) {
    const bool is_k = i >= nq;
    int head, u;
    if (is_k) {
      head = (i - nq) / (nrot + npass);
      u = (i - nq) - head * (nrot + npass);
    } else {
      head = i / nrot;
      u = i - head * nrot;
    }
    T* src = row + (size_t)(is_k ? H + head : head) * dk;
    const size_t krow = ((size_t)blk * G + head) * block_size + off;
    T* dst = is_k ? k_cache + krow * dk : src;
    T* vdst = is_k && shared ? v_cache + krow * dv : nullptr;
    P a;
    if (u >= nrot) {                                 // key dims that do not rotate
      const int e = rd + (u - nrot) * C;
      a.load(src + e);
      a.store_raw(dst + e);
      if (vdst) a.store_raw(vdst + e);
    } else if constexpr (PAIR) {
      const int e0 = HALF ? u * C : 2 * u, e1 = HALF ? e0 + rh : 2 * u + 1;
      P b;
      a.load(src + e0);
      b.load(src + e1);
      float x[C], y[C];
#pragma unroll
      for (int j = 0; j < C; ++j) {
        const int p = HALF ? e0 + j : u;
        const float c = cs[p], sn = cs[rh + p];
        x[j] = a.f[j] * c - b.f[j] * sn;
        y[j] = b.f[j] * c + a.f[j] * sn;
      }
      P::store(dst + e0, x);
      P::store(dst + e1, y);
      if (vdst) {
        a.store_raw(vdst + e0);
        b.store_raw(vdst + e1);
      }
    } else {
      const int e0 = u * C;
      a.load(src + e0);
      float x[C];
#pragma unroll
      for (int j = 0; j + 1 < C; j += 2) {
        const int p = (e0 + j) >> 1;
        const float c = cs[p], sn = cs[rh + p];
        x[j] = a.f[j] * c - a.f[j + 1] * sn;
        x[j + 1] = a.f[j + 1] * c + a.f[j] * sn;
      }
      P::store(dst + e0, x);
      if (vdst) a.store_raw(vdst + e0);
    }
  }
  if (slot >= 0 && !shared) {
    const T* vsrc = row + (size_t)(H + G) * dk;
    const int cpv = dv / C;
    for (int i = threadIdx.x; i < G * cpv; i += 256) {
      const int head = i / cpv, c = i - head * cpv;
      P a;
      a.load(vsrc + (size_t)head * dv + c * C);
      a.store_raw(v_cache + (((size_t)blk * G + head) * block_size + off) * dv + c * C);
    }
  }
}

}  // namespace

extern "C" int dgi_qk_rope(void* qkv, int is_f32, int T, int stride, const int* positions, const int* slots,
                           const float* cos_sin, int rd, int H, int G, int dk, int dv, void* k_cache, void* v_cache,
                           int block_size, int half, int shared, hipStream_t s) {
  if (T == 0) return 0;
  if (rd < 0 || rd > dk || (rd & 1) || (rd > 0 && !cos_sin)) return -2;
  if (H <= 0 || G <= 0 || (shared && dk != dv)) return -3;
  const int E = is_f32 ? 4 : 8;
  const bool vec = dk % E == 0 && dv % E == 0 && stride % E == 0 && rd % E == 0 && (!half || (rd / 2) % E == 0) &&
                   (((uintptr_t)qkv | (uintptr_t)k_cache | (uintptr_t)v_cache) & 15) == 0;
#define DGI_QKR(TT_, CC_, HH_)                                                                                     \
  qk_rope_kernel<TT_, CC_, HH_><<<T, 256, 0, s>>>((TT_*)qkv, stride, positions, slots, cos_sin, rd, H, G, dk, dv,  \
                                                  (TT_*)k_cache, (TT_*)v_cache, block_size, shared)
  if (is_f32) {
    if (vec) { if (half) DGI_QKR(float, 4, true); else DGI_QKR(float, 4, false); }
    else { if (half) DGI_QKR(float, 1, true); else DGI_QKR(float, 1, false); }
  } else {
    if (vec) { if (half) DGI_QKR(uint16_t, 8, true); else DGI_QKR(uint16_t, 8, false); }
    else { if (half) DGI_QKR(uint16_t, 1, true); else DGI_QKR(uint16_t, 1, false); }
  }
#undef DGI_QKR
  DGI_CHECK_LAUNCH();
  return 0;
}
