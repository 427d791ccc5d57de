// dgi/csrc/mix/masked_attention.hip — row-wise softmax attention over the paged KV pool for any
// head geometry, in bf16 or fp32, with a block ("chunk") mask and an output gate.
//
// decode_attention.hip and prefill_attention.hip are MFMA kernels for bf16 heads of 64 / 128
// dims whose keys and values share one size.  This kernel is the general form the other
// geometries run on (key size != value size, sizes that are no multiple of 16, fp32 caches)
// and the one both step phases share: every query row — a decode row or one row of a prompt
// portion — is one wave that walks its own visible keys
//
//     [first(p), p],   first(p) = floor(p / mask) * mask   (mask > 0: keys of the row's own block
//                                                            of `mask` positions, counted from
//                                                            position 0 of the sequence)
//                      first(p) = 0                          (mask == 0: plain causal)
//                      first(p) = max(0, p + mask + 1)       (mask < 0: the last -mask positions, a sliding window)
//
// straight from the cache (this step's keys are written before it runs), so the result does
// not depend on how the prompt was cut into steps or on what else is in the batch.
// Scores, the online softmax and the output accumulation are fp32; exp is the accurate expf.
// Optional distance bias: dist_bias[min(p - j, n_dist - 1)][head] (fp32, one row per distance, the
// last row for everything farther) is added to the scaled score of key j before the softmax.
// Optional head factors: the scaled score is multiplied by head_scale[head] (fp32, any sign).
// Optional soft cap: the scaled (and biased) score s becomes softcap * tanh(s / softcap).
// Optional sinks: exp(sinks[head]) joins the softmax denominator of that head (a logit that has no
// key and no value; it is neither scaled nor capped).
// Optional epilogue: out *= sigmoid(gate), element by element or one gate per head (`gate_heads`): the mixer's
// output gate, read from the same fused projection row as q.
//
// Wave layout: lane j scores key first + 64 i + j (a contiguous dk-vector per lane, 16-byte
// loads where dk allows); the 64 probabilities go through LDS and every lane accumulates the
// value dims d = lane + 64 c, so the V reads of one key are one coalesced row.
// grid = (rows, H), 64 threads.
#include <algorithm>
#include "../common.h"

using namespace dgi;

namespace {

template <typename T> __device__ __forceinline__ float ldf(const T* p);
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldf<uint16_t>(const uint16_t* p) { return bf16_to_f32(*p); }
template <typename T> __device__ __forceinline__ void stf(T* p, float v);
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void stf<uint16_t>(uint16_t* p, float v) { *p = f32_to_bf16(v); }

constexpr int MAXC = 8;       // value dims per lane: dv <= 64 * MAXC
constexpr int MAXDK = 512;    // query vector staged in LDS

__device__ __forceinline__ float dot_row(const float* __restrict__ qs, const float* __restrict__ k, int dk) {
  float acc = 0.f;
  if ((dk & 3) == 0) {
    for (int e = 0; e < dk; e += 4) {
      const float4 v = *reinterpret_cast<const float4*>(k + e);
      acc += qs[e] * v.x + qs[e + 1] * v.y + qs[e + 2] * v.z + qs[e + 3] * v.w;
    }
  } else {
    for (int e = 0; e < dk; ++e) acc += qs[e] * k[e];
  }
  return acc;
}

__device__ __forceinline__ float dot_row(const float* __restrict__ qs, const uint16_t* __restrict__ k, int dk) {
  float acc = 0.f;
  if ((dk & 7) == 0) {
    for (int e = 0; e < dk; e += 8) {
      float f[8];
      unpack8(*reinterpret_cast<const u32x4*>(k + e), f);
#pragma unroll
      for (int j = 0; j < 8; ++j) acc += qs[e + j] * f[j];
    }
  } else {
    for (int e = 0; e < dk; ++e) acc += qs[e] * bf16_to_f32(k[e]);
  }
  return acc;
}

template <typename T>
__global__ __launch_bounds__(64) void masked_attn_rows_kernel(
    const T* __restrict__ q, int q_stride, const T* __restrict__ k_cache, const T* __restrict__ v_cache,
    const int* __restrict__ block_tables, int bt_stride, const int* __restrict__ cu_seqlens, int n_seqs,
    const int* __restrict__ positions, int G, int dk, int dv, int bs, float scale, int mask,
    const T* __restrict__ gate, int gate_stride, T* __restrict__ out, int out_stride,
    const float* __restrict__ dist_bias, int n_dist, float softcap, const float* __restrict__ sinks,
    const float* __restrict__ head_scale, int gate_heads) {
  __shared__ float qs[MAXDK];
  __shared__ float ps[64];
  __shared__ long long vo[64];

  const int row = blockIdx.x, head = blockIdx.y, H = gridDim.y;
  const int lane = threadIdx.x;
  const int kvh = head / (H / G);
  // the row's sequence: row index itself (decode rows), or the portion holding it (cu_seqlens)
  int seq = row;
  if (cu_seqlens) {
    int lo = 0, hi = n_seqs - 1;
    while (lo < hi) {
      const int mid = (lo + hi + 1) >> 1;
      if (cu_seqlens[mid] <= row) lo = mid; else hi = mid - 1;
    }
    seq = lo;
  }
  const int* bt = block_tables + (size_t)seq * bt_stride;
  const int pos = positions[row];
  const int first = mask > 0 ? (pos / mask) * mask : (mask < 0 ? max(0, pos + mask + 1) : 0);

  const T* qp = q + (size_t)row * q_stride + (size_t)head * dk;
  for (int e = lane; e < dk; e += 64) qs[e] = ldf<T>(qp + e);
  __syncthreads();

  float m_run = -__builtin_inff(), l_run = 0.f;
  float o[MAXC];
#pragma unroll
  for (int c = 0; c < MAXC; ++c) o[c] = 0.f;
  const int nc = (dv + 63) >> 6;

  for (int k0 = first; k0 <= pos; k0 += 64) {
    const int key = k0 + lane;
    const bool ok = key <= pos;
    float s = -__builtin_inff();
    long long vbase = 0;
    if (ok) {
      const int blk = bt[key / bs];
      const long long slot = ((long long)blk * G + kvh) * bs + (key % bs);
      s = dot_row(qs, k_cache + slot * dk, dk) * scale;
      if (head_scale) s *= head_scale[head];
      if (dist_bias) s += dist_bias[(size_t)min(pos - key, n_dist - 1) * H + head];
      if (softcap > 0.f) s = softcap * tanhf(s / softcap);
      vbase = slot * dv;
    }
    const float m_new = fmaxf(m_run, wave_max(s));     // lane 0's key k0 is always visible: finite
    const float p = ok ? expf(s - m_new) : 0.f;
    const float corr = expf(m_run - m_new);            // first tile: exp(-inf) = 0
    l_run = l_run * corr + wave_sum(p);
    m_run = m_new;
    __syncthreads();                                   // previous tile's ps / vo fully read
    ps[lane] = p;
    vo[lane] = vbase;
    __syncthreads();
    const int n = min(64, pos - k0 + 1);
#pragma unroll
    for (int c = 0; c < MAXC; ++c) {
      if (c < nc) {
        const int d = lane + 64 * c;
        float acc = o[c] * corr;
        if (d < dv)
          for (int j = 0; j < n; ++j) acc += ps[j] * ldf<T>(v_cache + vo[j] + d);
        o[c] = acc;
      }
    }
  }
  float inv = 1.f / l_run;
  if (sinks) {
    // the sink logit joins the denominator only: out = o / (l + exp(sink - m)), with the larger of the two as reference
    const float sk = sinks[head], m2 = fmaxf(m_run, sk);
    const float f = expf(m_run - m2);
    inv = f / (l_run * f + expf(sk - m2));
  }
  T* op = out + (size_t)row * out_stride + (size_t)head * dv;
  const T* gp = gate ? gate + (size_t)row * gate_stride + (gate_heads ? (size_t)head : (size_t)head * dv) : nullptr;
#pragma unroll
  for (int c = 0; c < MAXC; ++c) {
    const int d = lane + 64 * c;
    if (c < nc && d < dv) {
      float v = o[c] * inv;
      if (gp) v *= 1.f / (1.f + expf(-ldf<T>(gate_heads ? gp : gp + d)));
      stf<T>(op + d, v);
    }
  }
}

// ---------------------------------------------------------------------------------------------
// Grouped kernel: one workgroup per (row, kv head) serves all R = H / G query heads of the group
// from ONE pass over the keys, with 16-byte cache reads.  Eight waves take 64-key tiles round
// robin; in a tile a 16-lane group owns one key at a time (lane c of the group its 16-byte chunk c,
// against the same chunk of the R queries in registers), so one wave instruction reads four whole K
// rows and a row's lines are fetched once; the scores and then the probabilities go through LDS,
// and the values are read the same way.
// Partial outputs are combined over the four lane groups by shuffles and over the waves in LDS.
// Needs dk, dv multiples of 8 (bf16) / 4 (fp32), H / G <= 8 and (H / G) * dv <= 1024.
// A step of few rows over many keys is cut into gridDim.z runs of a row's tiles (one workgroup each; a run may be
// empty): every run leaves its maximum, sum of weights and unnormalised output in part_ml / part_o, and
// masked_attn_reduce_kernel combines them, adds the sink and applies the gate.
constexpr int GNW = 8;        // waves per workgroup

// sum over the 16 lanes of a row (every lane gets it)
__device__ __forceinline__ float row16_total(float v) {
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x128, 0xf, 0xf, false));
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x124, 0xf, 0xf, false));
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x122, 0xf, 0xf, false));
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x121, 0xf, 0xf, false));
  return v;
}

template <typename T, int R, int VP>
__global__ __launch_bounds__(64 * GNW) void masked_attn_group_kernel(
    const T* __restrict__ q, int q_stride, const T* __restrict__ k_cache, const T* __restrict__ v_cache,
    const int* __restrict__ block_tables, int bt_stride, const int* __restrict__ cu_seqlens, int n_seqs,
    const int* __restrict__ positions, int H, int dk, int dv, int bs, float scale, int mask,
    const T* __restrict__ gate, int gate_stride, T* __restrict__ out, int out_stride,
    const float* __restrict__ dist_bias, int n_dist, float softcap, const float* __restrict__ sinks,
    const float* __restrict__ head_scale, int gate_heads, float* __restrict__ part_o, float* __restrict__ part_ml) {
  constexpr int E = 16 / sizeof(T);
  extern __shared__ __attribute__((aligned(16))) float smem[];
  const int row = blockIdx.x, kvh = blockIdx.y, G = gridDim.y;
  const int r = H / G;
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63;
  const int lg = lane >> 4, lc = lane & 15;
  float* qs = smem;                                  // [R][dk]
  float* ps = qs + R * dk;                           // [GNW][R][64]
  int* vs = reinterpret_cast<int*>(ps + GNW * R * 64);   // [GNW][64] cache slot of each key of the wave's tile
  float* cm = reinterpret_cast<float*>(vs + GNW * 64);   // [GNW][R] running max, then [GNW][R] sums
  float* co = cm + 2 * GNW * R;                      // [GNW][R][dv] partial outputs

  int seq = row;
  if (cu_seqlens) {
    int lo = 0, hi = n_seqs - 1;
    while (lo < hi) {
      const int mid = (lo + hi + 1) >> 1;
      if (cu_seqlens[mid] <= row) lo = mid; else hi = mid - 1;
    }
    seq = lo;
  }
  const int* bt = block_tables + (size_t)seq * bt_stride;
  const int pos = positions[row];
  const int first = mask > 0 ? (pos / mask) * mask : (mask < 0 ? max(0, pos + mask + 1) : 0);

  const T* qp = q + (size_t)row * q_stride + (size_t)kvh * r * dk;
  for (int e = tid; e < r * dk; e += 64 * GNW) qs[e] = ldf<T>(qp + e);
  __syncthreads();

  // this lane's chunks of the queries: in registers where they fit, else read from LDS again for every key
  constexpr bool QREG = R * VP * E <= 64;
  constexpr int U = VP == 1 ? 8 : 4;
  float qr[QREG ? R : 1][QREG ? VP : 1][E];
  if constexpr (QREG) {
#pragma unroll
    for (int i = 0; i < R; ++i)
#pragma unroll
      for (int p = 0; p < VP; ++p)
#pragma unroll
        for (int j = 0; j < E; ++j) {
          const int c = (lc + 16 * p) * E + j;
          qr[i][p][j] = i < r && c < dk ? qs[i * dk + c] : 0.f;
        }
  }
  float m[R], l[R], o[R][VP][E];
#pragma unroll
  for (int i = 0; i < R; ++i) {
    m[i] = -__builtin_inff();
    l[i] = 0.f;
#pragma unroll
    for (int p = 0; p < VP; ++p)
#pragma unroll
      for (int j = 0; j < E; ++j) o[i][p][j] = 0.f;
  }
  float* psw = ps + w * R * 64;
  int* vsw = vs + w * 64;
  const int ntiles = (pos - first) / 64 + 1;
  const int tpr = (ntiles + (int)gridDim.z - 1) / (int)gridDim.z;      // tiles per run
  const int t_end = min(ntiles, ((int)blockIdx.z + 1) * tpr);
  for (int tile = blockIdx.z * tpr + w; tile < t_end; tile += GNW) {
    const int k0 = first + tile * 64;
    const int key = k0 + lane;
    const bool ok = key <= pos;
    const int kq = min(key, pos);                        // lanes past the last key point at it: every load stays in bounds
    vsw[lane] = (bt[kq / bs] * G + kvh) * bs + (kq % bs);
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    const int n = min(64, pos - k0 + 1);
    // U keys per group at a time, all their rows requested before the first is used; places past n repeat the last key
    u32x4 raw[U][VP];
    auto load_rows = [&](const T* cache, int d, int kk0) {
      int sl[U];
#pragma unroll
      for (int u = 0; u < U; ++u) sl[u] = vsw[kk0 + 4 * u + lg];
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int p = 0; p < VP; ++p) {
          const int c = (lc + 16 * p) * E;
          raw[u][p] = c < d ? *reinterpret_cast<const u32x4*>(cache + (size_t)sl[u] * d + c) : u32x4{0u, 0u, 0u, 0u};
        }
    };
    auto as_floats = [&](const u32x4& v, float* f) {
      if constexpr (sizeof(T) == 2) {
        unpack8(v, f);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j) f[j] = __uint_as_float(v[j]);
      }
    };
    for (int kk0 = 0; kk0 < n; kk0 += 4 * U) {
      load_rows(k_cache, dk, kk0);
#pragma unroll
      for (int u = 0; u < U; ++u) {
        float acc[R];
#pragma unroll
        for (int i = 0; i < R; ++i) acc[i] = 0.f;
#pragma unroll
        for (int p = 0; p < VP; ++p) {
          float kf[E];
          as_floats(raw[u][p], kf);
          const int c = (lc + 16 * p) * E;
#pragma unroll
          for (int i = 0; i < R; ++i) {
            if constexpr (QREG) {
#pragma unroll
              for (int j = 0; j < E; ++j) acc[i] += qr[i][p][j] * kf[j];
            } else if (i < r && c < dk) {
#pragma unroll
              for (int j = 0; j < E; ++j) acc[i] += qs[i * dk + c + j] * kf[j];
            }
          }
        }
        float mine = 0.f;                                // lane i of the group keeps head i's score
#pragma unroll
        for (int i = 0; i < R; ++i) {
          const float tot = row16_total(acc[i]);
          mine = lc == i ? tot : mine;
        }
        if (lc < R) psw[lc * 64 + kk0 + 4 * u + lg] = mine;
      }
    }
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll
    for (int i = 0; i < R; ++i) {
      if (i < r) {
        float s = -__builtin_inff();
        if (ok) {
          s = psw[i * 64 + lane] * scale;
          if (head_scale) s *= head_scale[kvh * r + i];
          if (dist_bias) s += dist_bias[(size_t)min(pos - key, n_dist - 1) * H + kvh * r + i];
          if (softcap > 0.f) s = softcap * tanhf(s / softcap);
        }
        const float m_new = fmaxf(m[i], wave_max(s));       // key k0 (lane 0) is visible: finite
        const float p = ok ? expf(s - m_new) : 0.f;
        const float corr = expf(m[i] - m_new);
        l[i] = l[i] * corr + wave_sum(p);
        m[i] = m_new;
#pragma unroll
        for (int vp = 0; vp < VP; ++vp)
#pragma unroll
          for (int j = 0; j < E; ++j) o[i][vp][j] *= corr;
        psw[i * 64 + lane] = p;                          // over the lane's own score
      }
    }
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    for (int kk0 = 0; kk0 < n; kk0 += 4 * U) {
      load_rows(v_cache, dv, kk0);
#pragma unroll
      for (int u = 0; u < U; ++u) {
        float pk[R];                                     // 0 past n
#pragma unroll
        for (int i = 0; i < R; ++i) pk[i] = i < r ? psw[i * 64 + kk0 + 4 * u + lg] : 0.f;
#pragma unroll
        for (int vp = 0; vp < VP; ++vp) {
          float vf[E];
          as_floats(raw[u][vp], vf);
#pragma unroll
          for (int i = 0; i < R; ++i)
#pragma unroll
            for (int j = 0; j < E; ++j) o[i][vp][j] += pk[i] * vf[j];
        }
      }
    }
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  // lane groups -> lane group 0, then waves -> LDS
#pragma unroll
  for (int i = 0; i < R; ++i)
#pragma unroll
    for (int vp = 0; vp < VP; ++vp)
#pragma unroll
      for (int j = 0; j < E; ++j) {
        float v = o[i][vp][j];
        v += __shfl_xor(v, 16, 64);
        v += __shfl_xor(v, 32, 64);
        o[i][vp][j] = v;
      }
  if (lane == 0) {
#pragma unroll
    for (int i = 0; i < R; ++i) {
      cm[w * R + i] = m[i];
      cm[GNW * R + w * R + i] = l[i];
    }
  }
  if (lg == 0) {
#pragma unroll
    for (int i = 0; i < R; ++i)
      if (i < r)
#pragma unroll
        for (int vp = 0; vp < VP; ++vp) {
          const int c = (lc + 16 * vp) * E;
          if (c < dv)
#pragma unroll
            for (int j = 0; j < E; ++j) co[((size_t)w * R + i) * dv + c + j] = o[i][vp][j];
        }
  }
  __syncthreads();
  for (int idx = tid; idx < r * dv; idx += 64 * GNW) {
    const int i = idx / dv, d = idx - i * dv;
    const int head = kvh * r + i;
    if (part_o) {
      float M = -__builtin_inff(), L = 0.f, O = 0.f;
#pragma unroll
      for (int ww = 0; ww < GNW; ++ww) M = fmaxf(M, cm[ww * R + i]);
      if (M != -__builtin_inff()) {                    // an empty run leaves zeros
#pragma unroll
        for (int ww = 0; ww < GNW; ++ww) {
          const float f = expf(cm[ww * R + i] - M);
          L += cm[GNW * R + ww * R + i] * f;
          O += co[((size_t)ww * R + i) * dv + d] * f;
        }
      }
      const size_t slot = ((size_t)blockIdx.z * gridDim.x + row) * H + head;
      part_o[slot * dv + d] = O;
      if (d == 0) {
        part_ml[2 * slot] = M;
        part_ml[2 * slot + 1] = L;
      }
      continue;
    }
    float M = sinks ? sinks[head] : -__builtin_inff();
#pragma unroll
    for (int ww = 0; ww < GNW; ++ww) M = fmaxf(M, cm[ww * R + i]);
    float L = sinks ? expf(sinks[head] - M) : 0.f, O = 0.f;      // the sink: one more term of the denominator
#pragma unroll
    for (int ww = 0; ww < GNW; ++ww) {
      const float f = expf(cm[ww * R + i] - M);          // waves without a tile: exp(-inf) = 0
      L += cm[GNW * R + ww * R + i] * f;
      O += co[((size_t)ww * R + i) * dv + d] * f;
    }
    float v = O / L;
    if (gate) v *= 1.f / (1.f + expf(-ldf<T>(gate + (size_t)row * gate_stride + (gate_heads ? (size_t)head : (size_t)head * dv + d))));
    stf<T>(out + (size_t)row * out_stride + (size_t)head * dv + d, v);
  }
}

// combines the runs of masked_attn_group_kernel; grid (rows, H)
template <typename T>
__global__ __launch_bounds__(128) void masked_attn_reduce_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml,
                                                                 int nsplit, int dv, const float* __restrict__ sinks,
                                                                 const T* __restrict__ gate, int gate_stride, int gate_heads,
                                                                 T* __restrict__ out, int out_stride) {
  const int row = blockIdx.x, head = blockIdx.y, rows = gridDim.x, H = gridDim.y;
  float M = sinks ? sinks[head] : -__builtin_inff();
  for (int z = 0; z < nsplit; ++z) M = fmaxf(M, part_ml[2 * (((size_t)z * rows + row) * H + head)]);     // run 0 is never empty
  float L = sinks ? expf(sinks[head] - M) : 0.f;
  for (int z = 0; z < nsplit; ++z) {
    const size_t slot = ((size_t)z * rows + row) * H + head;
    L += part_ml[2 * slot + 1] * expf(part_ml[2 * slot] - M);
  }
  const float inv = 1.f / L;
  for (int d = threadIdx.x; d < dv; d += 128) {
    float O = 0.f;
    for (int z = 0; z < nsplit; ++z) {
      const size_t slot = ((size_t)z * rows + row) * H + head;
      O += part_o[slot * dv + d] * expf(part_ml[2 * slot] - M);
    }
    float v = O * inv;
    if (gate) v *= 1.f / (1.f + expf(-ldf<T>(gate + (size_t)row * gate_stride + (gate_heads ? (size_t)head : (size_t)head * dv + d))));
    stf<T>(out + (size_t)row * out_stride + (size_t)head * dv + d, v);
  }
}

template <typename T, int R, int VP>
int launch_group(const void* q, int q_stride, const void* k_cache, const void* v_cache, const int* block_tables,
                 int bt_stride, const int* cu_seqlens, int n_seqs, const int* positions, int rows, int H, int G, int dk,
                 int dv, int bs, float scale, int mask, const void* gate, int gate_stride, void* out, int out_stride,
                 const float* dist_bias, int n_dist, float softcap, const float* sinks, const float* head_scale, int gate_heads,
                 int nsplit, float* part_o, float* part_ml, hipStream_t s) {
  const size_t lds = (size_t)(R * dk + GNW * R * 64 + GNW * 64 + 2 * GNW * R + GNW * R * dv) * 4;
  if (lds > 64 * 1024) return -1;
  if (nsplit < 2) part_o = part_ml = nullptr;
  masked_attn_group_kernel<T, R, VP><<<dim3(rows, G, nsplit), 64 * GNW, lds, s>>>(
      (const T*)q, q_stride, (const T*)k_cache, (const T*)v_cache, block_tables, bt_stride, cu_seqlens, n_seqs,
      positions, H, dk, dv, bs, scale, mask, (const T*)gate, gate_stride, (T*)out, out_stride, dist_bias, n_dist,
      softcap, sinks, head_scale, gate_heads, part_o, part_ml);
  if (nsplit > 1)
    masked_attn_reduce_kernel<T><<<dim3(rows, H), 128, 0, s>>>(part_o, part_ml, nsplit, dv, sinks, (const T*)gate, gate_stride,
                                                               gate_heads, (T*)out, out_stride);
  return 0;
}

template <typename T>
int dispatch_group(int r, int vpn, const void* q, int q_stride, const void* k_cache, const void* v_cache,
                   const int* block_tables, int bt_stride, const int* cu_seqlens, int n_seqs, const int* positions,
                   int rows, int H, int G, int dk, int dv, int bs, float scale, int mask, const void* gate,
                   int gate_stride, void* out, int out_stride, const float* dist_bias, int n_dist, float softcap,
                   const float* sinks, const float* head_scale, int gate_heads, int nsplit, float* part_o, float* part_ml, hipStream_t s) {
#define DGI_GRP(RV, VPV)                                                                                       \
  return launch_group<T, RV, VPV>(q, q_stride, k_cache, v_cache, block_tables, bt_stride, cu_seqlens, n_seqs, \
                                  positions, rows, H, G, dk, dv, bs, scale, mask, gate, gate_stride, out, out_stride, dist_bias, \
                                  n_dist, softcap, sinks, head_scale, gate_heads, nsplit, part_o, part_ml, s)
  if (vpn == 1) {
    if (r == 1) DGI_GRP(1, 1);
    if (r == 2) DGI_GRP(2, 1);
    if (r <= 4) DGI_GRP(4, 1);
    DGI_GRP(8, 1);
  }
  if (r == 1) DGI_GRP(1, 2);
  if (r == 2) DGI_GRP(2, 2);
  if (r <= 4) DGI_GRP(4, 2);
  DGI_GRP(8, 2);
#undef DGI_GRP
}

}  // namespace

// q / gate / out: row-major with their own row strides (elements); cu_seqlens (n_seqs + 1 row
// offsets) maps rows to block-table rows, nullptr: row i uses block-table row i.  nsplit > 1: runs of keys per row for
// the grouped kernel (the other one takes a row in one go), with part_o [nsplit, rows, H, dv] and part_ml
// [nsplit, rows, H, 2] fp32 to meet in.
extern "C" int dgi_masked_attn_rows(const void* q, int q_stride, const void* k_cache, const void* v_cache,
                                    const int* block_tables, int bt_stride, const int* cu_seqlens, int n_seqs,
                                    const int* positions, int rows, int H, int G, int dk, int dv, int block_size,
                                    float scale, int mask, const void* gate, int gate_stride, void* out,
                                    int out_stride, int is_f32, const float* dist_bias, int n_dist, float softcap,
                                    const float* sinks, const float* head_scale, int gate_heads, int nsplit, float* part_o,
                                    float* part_ml, hipStream_t s) {
  if (rows == 0) return 0;
  if (G <= 0 || H % G) return -2;
  if (dk > MAXDK || dv > 64 * MAXC || dk <= 0 || dv <= 0) return -3;
  if (H > 65535) return -4;
  if (nsplit < 1 || nsplit > 65535 || (nsplit > 1 && (!part_o || !part_ml))) return -6;
  if (dist_bias && n_dist < 1) return -5;
  {
    // grouped kernel where the geometry allows (see masked_attn_group_kernel)
    const int E = is_f32 ? 4 : 8, r = H / G;
    const int vpn = (std::max(dk, dv) + 16 * E - 1) / (16 * E);
    const bool aligned = ((uintptr_t)k_cache | (uintptr_t)v_cache) % 16 == 0;
    if (dk % E == 0 && dv % E == 0 && r <= 8 && vpn <= 2 && r * dv <= 1024 && aligned && G <= 65535) {
      const int rc = is_f32 ? dispatch_group<float>(r, vpn, q, q_stride, k_cache, v_cache, block_tables, bt_stride, cu_seqlens,
                                                    n_seqs, positions, rows, H, G, dk, dv, block_size, scale, mask, gate,
                                                    gate_stride, out, out_stride, dist_bias, n_dist, softcap, sinks, head_scale,
                                                    gate_heads, nsplit, part_o, part_ml, s)
                            : dispatch_group<uint16_t>(r, vpn, q, q_stride, k_cache, v_cache, block_tables, bt_stride,
                                                       cu_seqlens, n_seqs, positions, rows, H, G, dk, dv, block_size, scale,
                                                       mask, gate, gate_stride, out, out_stride, dist_bias, n_dist, softcap,
                                                       sinks, head_scale, gate_heads, nsplit, part_o, part_ml, s);
      if (rc == 0) {
        DGI_CHECK_LAUNCH();
        return 0;
      }
    }
  }
  const dim3 grid(rows, H);
  if (is_f32)
    masked_attn_rows_kernel<float><<<grid, 64, 0, s>>>(
        (const float*)q, q_stride, (const float*)k_cache, (const float*)v_cache, block_tables, bt_stride, cu_seqlens,
        n_seqs, positions, G, dk, dv, block_size, scale, mask, (const float*)gate, gate_stride, (float*)out, out_stride,
        dist_bias, n_dist, softcap, sinks, head_scale, gate_heads);
  else
    masked_attn_rows_kernel<uint16_t><<<grid, 64, 0, s>>>(
        (const uint16_t*)q, q_stride, (const uint16_t*)k_cache, (const uint16_t*)v_cache, block_tables, bt_stride,
        cu_seqlens, n_seqs, positions, G, dk, dv, block_size, scale, mask, (const uint16_t*)gate, gate_stride,
        (uint16_t*)out, out_stride, dist_bias, n_dist, softcap, sinks, head_scale, gate_heads);
  DGI_CHECK_LAUNCH();
  return 0;
}
