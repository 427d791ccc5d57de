// dgi/csrc/mix/chunk_scan.hip — linear_scan's decayed recurrences (gla, light: see linear_scan.hip) for prompt portions, sixteen
// tokens at a time in fp32 matrix products (v_mfma_f32_16x16x4_f32):
//
//     S_t = diag(a_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t                       S [dk, dv] fp32
//
// With b_t the product of the decays of the chunk's tokens up to t (per key channel) and b the product of all sixteen,
//
//     o_t = (q_t b_t)^T S + sum_(s <= t) [(q_t b_t) . (k_s / b_s)] v_s,        S <- diag(b) S + sum_s (k_s b / b_s) v_s^T
//
// A workgroup owns (sequence, head, 16 value columns).  Four waves compute: wave w holds the state rows of the 16-channel
// tiles w, w + 4, .. in registers, in the layout the products leave them (the key index inside a product is permuted so that the
// state registers are its operand as they are).  The waves' partial score tiles and outputs meet in LDS.  Four more
// waves prepare: wave w loads the same channels of the next chunk, forms the running products and writes the scaled
// operands to the other LDS buffer, and stores the previous chunk's outputs.  Their loads run NP chunks ahead in a register
// ring (the chunk loop is unrolled NP times).  Two barriers per chunk.
//
// Products of decays can leave the fp32 range.  A wave whose channels decay by more than 1e28 within a chunk gets the raw
// values instead and runs that chunk token by token on the same registers (its contribution to the outputs is a
// sum over its own channels, so waves may differ).  A portion at position 0 reads no state.
#include <type_traits>
#include "../common.h"

using namespace dgi;

namespace {

template <typename T> __device__ __forceinline__ float ldf(const T* p);
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldf<uint16_t>(const uint16_t* p) { return bf16_to_f32(*p); }

constexpr int C = 16;              // tokens per chunk
constexpr int TR = 20;             // padded row of sixteen tokens
constexpr float SAFE = 1e-28f;

struct ChunkArgs {
  float* y;
  const void *q, *k, *v;
  int q_stride, k_stride, v_stride;
  const float* decay;              // per channel: [T, H * dk]; per head: [H]
  int decay_stride;
  float* state;
  const int *positions, *seq_row0, *seq_slots;
  int H, dk, dv;
};

__device__ __forceinline__ float4 ld4(const float* p) { return *reinterpret_cast<const float4*>(p); }

// LIGHT: one decay per head and SiLU on q, k, v; else a decay per token and channel and q scaled by dk^-1/2.
// TD: 16-channel tiles per wave (dk <= 64 TD)
template <bool LIGHT, typename TI, int TD>
__global__ __launch_bounds__(512) void chunk_scan_kernel(const ChunkArgs a) {
  constexpr int DP = 64 * TD, QR = DP + 4;
  constexpr int BUF = 2 * C * QR + DP * TR + C * TR + DP + 4;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* redA = sm + 2 * BUF;      // [4][16][17]
  float* redO = redA + 4 * 16 * 17 + 4;      // [4][16][16]
  const int seq = blockIdx.x, head = blockIdx.y, col0 = blockIdx.z * 16;
  const int row0 = a.seq_row0[seq], n = a.seq_row0[seq + 1] - row0;
  if (n <= 0) return;
  const int p0 = a.positions[row0], slot = a.seq_slots[seq];
  const int H = a.H, dk = a.dk, dv = a.dv;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int n16 = lane & 15, g = lane >> 4;
  const bool computes = wave < 4;
  const int w = wave & 3;
  const int chunks = (n + C - 1) / C;
  const float qscale = LIGHT ? 1.f : 1.f / sqrtf((float)dk);
  const float hdecay = LIGHT ? a.decay[head] : 0.f;

  auto Qs = [&](int b) { return sm + b * BUF; };                             // [16][QR]   q b_t
  auto Ks = [&](int b) { return sm + b * BUF + C * QR; };                    // [16][QR]   k / b_t
  auto KT = [&](int b) { return sm + b * BUF + 2 * C * QR; };                // [DP][TR]   k b / b_t by channel (raw chunk: decays)
  auto VT = [&](int b) { return sm + b * BUF + 2 * C * QR + DP * TR; };      // [16][TR]   v by column
  auto Bc = [&](int b) { return sm + b * BUF + 2 * C * QR + DP * TR + C * TR; };      // [DP]
  auto Raw = [&](int b) { return sm + b * BUF + 2 * C * QR + DP * TR + C * TR + DP; };      // [4] wave runs the chunk raw

  // ---- preparing waves: lane = (channel n16 of the tile, tokens 4 g ..)
  constexpr int NP = TD == 1 ? 4 : (TD == 2 ? 2 : 1);
  // kept as loaded: a conversion at the load would wait for it on the spot
  TI rq[NP][TD][4], rk[NP][TD][4], rv[NP];
  float rd[NP][TD][4];
  const TI* qb = (const TI*)a.q + (size_t)row0 * a.q_stride + head * dk;
  const TI* kb = (const TI*)a.k + (size_t)row0 * a.k_stride + head * dk;
  const TI* vb = (const TI*)a.v + (size_t)row0 * a.v_stride + (size_t)head * dv + col0;
  const float* db = LIGHT ? nullptr : a.decay + (size_t)row0 * a.decay_stride + head * dk;
  // loads run unconditionally (rows and channels clamped into the portion); prepare() drops what is outside
  auto load = [&](int ci, int st) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = min(ci * C + 4 * g + i, n - 1);
#pragma unroll
      for (int td = 0; td < TD; ++td) {
        const int ch = min(16 * (td * 4 + w) + n16, dk - 1);
        rq[st][td][i] = qb[(size_t)t * a.q_stride + ch];
        rk[st][td][i] = kb[(size_t)t * a.k_stride + ch];
        if constexpr (!LIGHT) rd[st][td][i] = db[(size_t)t * a.decay_stride + ch];
      }
    }
    rv[st] = vb[(size_t)min(ci * C + 4 * w + g, n - 1) * a.v_stride + min(n16, dv - 1 - col0)];
  };
  auto silu = [](float x) {
    return x * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(x * -1.4426950408889634f));
  };
  auto prepare = [&](int ci, int st) {
    const int b = ci & 1, left = n - ci * C;         // tokens from this chunk on
    float q[TD][4], k[TD][4], d[TD][4], bt[TD][4], tot[TD];
    bool raw = false;
#pragma unroll
    for (int td = 0; td < TD; ++td) {
      const bool in = 16 * (td * 4 + w) + n16 < dk;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const bool ok = in && 4 * g + i < left;
        q[td][i] = ok ? ldf<TI>(&rq[st][td][i]) : 0.f;
        k[td][i] = ok ? ldf<TI>(&rk[st][td][i]) : 0.f;
        if constexpr (LIGHT) d[td][i] = ok ? hdecay : 1.f;
        else d[td][i] = ok ? rd[st][td][i] : 1.f;
      }
    }
    const float v = (4 * w + g < left && col0 + n16 < dv) ? ldf<TI>(&rv[st]) : 0.f;
#pragma unroll
    for (int td = 0; td < TD; ++td) {
      bt[td][0] = d[td][0];
#pragma unroll
      for (int i = 1; i < 4; ++i) bt[td][i] = bt[td][i - 1] * d[td][i];
      const float p = bt[td][3];
      const float p0_ = __shfl(p, n16, 64), p1_ = __shfl(p, n16 + 16, 64), p2_ = __shfl(p, n16 + 32, 64), p3_ = __shfl(p, n16 + 48, 64);
      const float e = (g > 0 ? p0_ : 1.f) * (g > 1 ? p1_ : 1.f) * (g > 2 ? p2_ : 1.f);
      tot[td] = p0_ * p1_ * p2_ * p3_;
#pragma unroll
      for (int i = 0; i < 4; ++i) bt[td][i] *= e;
      raw |= !(tot[td] > SAFE);
    }
    raw = __any(raw);
#pragma unroll
    for (int td = 0; td < TD; ++td) {
      const int ch = 16 * (td * 4 + w) + n16;
      float kt[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        float qi = LIGHT ? silu(q[td][i]) : q[td][i] * qscale, ki = LIGHT ? silu(k[td][i]) : k[td][i];
        if (raw) {
          kt[i] = d[td][i];
        } else {
          qi *= bt[td][i];
          ki *= __builtin_amdgcn_rcpf(bt[td][i]);
          kt[i] = ki * tot[td];
        }
        Qs(b)[(4 * g + i) * QR + ch] = qi;
        Ks(b)[(4 * g + i) * QR + ch] = ki;
      }
      *reinterpret_cast<float4*>(KT(b) + ch * TR + 4 * g) = make_float4(kt[0], kt[1], kt[2], kt[3]);
      if (g == 0) Bc(b)[ch] = tot[td];
    }
    VT(b)[n16 * TR + 4 * w + g] = LIGHT ? silu(v) : v;
    if (lane == 0) Raw(b)[w] = raw ? 1.f : 0.f;
  };
  auto store = [&](int ci) {       // outputs of chunk ci: one per lane of the preparing waves
    const int t = 4 * w + g, col = col0 + n16;
    const float* r = redO + t * 16 + n16;
    const float o = (r[0] + r[256]) + (r[512] + r[768]);
    if (ci * C + t < n && col < dv) a.y[(size_t)(row0 + ci * C + t) * H * dv + (size_t)head * dv + col] = o;
  };

  // The two roles run loops of their own (a wave never changes its role) with the same barriers: two per chunk, one before.
  if (!computes) {
    const int last = chunks - 1;
#pragma unroll
    for (int st = 0; st < NP; ++st) load(min(st, last), st);
    prepare(0, 0);
    load(min(NP, last), 0);
    __syncthreads();
    // st: the chunk's place in the register ring (its index modulo NP)
    auto step = [&](int ci, auto stage) {
      constexpr int nx = (decltype(stage)::value + 1) % NP;
      if (ci > 0) store(ci - 1);
      if (ci < last) {
        prepare(ci + 1, nx);
        load(min(ci + 1 + NP, last), nx);
      }
      __syncthreads();
      __syncthreads();
    };
    for (int ci = 0; ci < chunks; ci += NP) {
      step(ci, std::integral_constant<int, 0>{});
      if constexpr (NP > 1) {
        if (ci + 1 < chunks) step(ci + 1, std::integral_constant<int, 1>{});
      }
      if constexpr (NP > 2) {
        if (ci + 2 < chunks) step(ci + 2, std::integral_constant<int, 2>{});
        if (ci + 3 < chunks) step(ci + 3, std::integral_constant<int, 3>{});
      }
    }
    store(last);
    return;
  }

  // ---- computing waves: state rows 4 g + r of the wave's tiles, column n16
  f32x4 S[TD];
  const int col = col0 + n16;
  const size_t sbase = ((size_t)slot * H + head) * dk;
#pragma unroll
  for (int td = 0; td < TD; ++td)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int ch = 16 * (td * 4 + w) + 4 * g + r;
      S[td][r] = (p0 > 0 && ch < dk && col < dv) ? a.state[(sbase + ch) * dv + col] : 0.f;
    }
  __syncthreads();
  for (int ci = 0; ci < chunks; ++ci) {
    const int b = ci & 1;
    f32x4 accO = {0.f, 0.f, 0.f, 0.f};
    f32x4 accA = {0.f, 0.f, 0.f, 0.f};
    if (Raw(b)[w] == 0.f) {
      const float4 vf = ld4(VT(b) + n16 * TR + 4 * g);
#pragma unroll
      for (int td = 0; td < TD; ++td) {
        const int ch0 = 16 * (td * 4 + w);
        const float4 qf = ld4(Qs(b) + n16 * QR + ch0 + 4 * g), kf = ld4(Ks(b) + n16 * QR + ch0 + 4 * g);
        const float4 kt = ld4(KT(b) + (ch0 + n16) * TR + 4 * g), bc = ld4(Bc(b) + ch0 + 4 * g);
        f32x4 u = S[td];
        accA = __builtin_amdgcn_mfma_f32_16x16x4f32(qf.x, kf.x, accA, 0, 0, 0);
        accO = __builtin_amdgcn_mfma_f32_16x16x4f32(qf.x, u[0], accO, 0, 0, 0);
        accA = __builtin_amdgcn_mfma_f32_16x16x4f32(qf.y, kf.y, accA, 0, 0, 0);
        accO = __builtin_amdgcn_mfma_f32_16x16x4f32(qf.y, u[1], accO, 0, 0, 0);
        accA = __builtin_amdgcn_mfma_f32_16x16x4f32(qf.z, kf.z, accA, 0, 0, 0);
        accO = __builtin_amdgcn_mfma_f32_16x16x4f32(qf.z, u[2], accO, 0, 0, 0);
        accA = __builtin_amdgcn_mfma_f32_16x16x4f32(qf.w, kf.w, accA, 0, 0, 0);
        accO = __builtin_amdgcn_mfma_f32_16x16x4f32(qf.w, u[3], accO, 0, 0, 0);
        u[0] *= bc.x; u[1] *= bc.y; u[2] *= bc.z; u[3] *= bc.w;
        u = __builtin_amdgcn_mfma_f32_16x16x4f32(kt.x, vf.x, u, 0, 0, 0);
        u = __builtin_amdgcn_mfma_f32_16x16x4f32(kt.y, vf.y, u, 0, 0, 0);
        u = __builtin_amdgcn_mfma_f32_16x16x4f32(kt.z, vf.z, u, 0, 0, 0);
        u = __builtin_amdgcn_mfma_f32_16x16x4f32(kt.w, vf.w, u, 0, 0, 0);
        S[td] = u;
      }
    } else {
#pragma unroll
      for (int t = 0; t < C; ++t) {
        const float vj = VT(b)[n16 * TR + t];
        float o = 0.f;
#pragma unroll
        for (int td = 0; td < TD; ++td) {
          const int c4 = 16 * (td * 4 + w) + 4 * g;
          const float4 qf = ld4(Qs(b) + t * QR + c4), kf = ld4(Ks(b) + t * QR + c4);
          const float* al = KT(b) + c4 * TR + t;
          S[td][0] = al[0] * S[td][0] + kf.x * vj;
          S[td][1] = al[TR] * S[td][1] + kf.y * vj;
          S[td][2] = al[2 * TR] * S[td][2] + kf.z * vj;
          S[td][3] = al[3 * TR] * S[td][3] + kf.w * vj;
          o += S[td][0] * qf.x + S[td][1] * qf.y + S[td][2] * qf.z + S[td][3] * qf.w;
        }
        o += __shfl_xor(o, 16, 64);
        o += __shfl_xor(o, 32, 64);
        if (g == (t >> 2)) accO[t & 3] = o;
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) redA[(w * 16 + 4 * g + r) * 17 + n16] = accA[r];
    __syncthreads();
    // scores of key token 4 w + g for query token n16, all channels; keys up to the query
    const int s = 4 * w + g;
    const float* r = redA + n16 * 17 + s;
    const float p = s <= n16 ? (r[0] + r[16 * 17]) + (r[2 * 16 * 17] + r[3 * 16 * 17]) : 0.f;
    accO = __builtin_amdgcn_mfma_f32_16x16x4f32(p, VT(b)[n16 * TR + s], accO, 0, 0, 0);
#pragma unroll
    for (int i = 0; i < 4; ++i) redO[w * 256 + (4 * g + i) * 16 + n16] = accO[i];
    __syncthreads();
  }
#pragma unroll
  for (int td = 0; td < TD; ++td)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int ch = 16 * (td * 4 + w) + 4 * g + r;
      if (ch < dk && col < dv) a.state[(sbase + ch) * dv + col] = S[td][r];
    }
}

template <bool LIGHT, typename TI, int TD>
int launch_one(const ChunkArgs& a, dim3 grid, hipStream_t st) {
  constexpr int DP = 64 * TD;
  constexpr size_t lds = (size_t)(2 * (2 * C * (DP + 4) + DP * TR + C * TR + DP + 4) + 4 * 16 * 17 + 4 + 4 * 256) * 4;
  static_assert(lds <= 160 * 1024, "LDS");
  auto kernel = chunk_scan_kernel<LIGHT, TI, TD>;
  if (lds > 64 * 1024) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return (int)e;
  }
  kernel<<<grid, 512, lds, st>>>(a);
  return 0;
}

template <bool LIGHT, typename TI>
int launch_dims(const ChunkArgs& a, dim3 grid, hipStream_t st) {
  if (a.dk <= 64) return launch_one<LIGHT, TI, 1>(a, grid, st);
  if (a.dk <= 128) return launch_one<LIGHT, TI, 2>(a, grid, st);
  return launch_one<LIGHT, TI, 4>(a, grid, st);
}

}  // namespace

// light: decay [H] and SiLU on q / k / v; else decay [T, H * dk] rows with their stride.  dk at most 256.
extern "C" int dgi_chunk_scan(float* y, int light, const void* q, int q_stride, const void* k, int k_stride, const void* v,
                              int v_stride, int in_f32, const float* decay, int decay_stride, float* state,
                              const int* positions, const int* seq_row0, const int* seq_slots, int n_seq, int H, int dk, int dv,
                              hipStream_t st) {
  if (n_seq == 0) return 0;
  if (dk <= 0 || dk > 256 || dv <= 0 || H <= 0 || H > 65535 || (dv + 15) / 16 > 65535 || !decay) return -3;
  ChunkArgs a;
  a.y = y; a.q = q; a.k = k; a.v = v;
  a.q_stride = q_stride; a.k_stride = k_stride; a.v_stride = v_stride;
  a.decay = decay; a.decay_stride = decay_stride; a.state = state;
  a.positions = positions; a.seq_row0 = seq_row0; a.seq_slots = seq_slots;
  a.H = H; a.dk = dk; a.dv = dv;
  const dim3 grid(n_seq, H, (dv + 15) / 16);
  int rc;
  if (light) rc = in_f32 ? launch_dims<true, float>(a, grid, st) : launch_dims<true, uint16_t>(a, grid, st);
  else rc = in_f32 ? launch_dims<false, float>(a, grid, st) : launch_dims<false, uint16_t>(a, grid, st);
  if (rc) return rc;
  DGI_CHECK_LAUNCH();
  return 0;
}
