// dgi/csrc/mix/sigmoid_attention.hip — attention over the paged KV pool whose heads' scores are mixed and whose weights
// are sigmoids, row by row, for any head geometry in bf16 or fp32:
//
//     s_g(j)  = scale * q_g . k_j                                    raw score of head g, key j
//     w_h(j)  = sigmoid(sum_g talk[h, g] s_g(j) + pb[h])             j in [first(p), p]
//     out_h   = sum_j w_h(j) v_j
//
// first(p) = max(0, p - window + 1) (window > 0: the last `window` positions, itself included), else 0.  Nothing is
// normalised over keys, so the sums of different runs of keys just add up.  talk == nullptr: every head its own
// score; pb == nullptr: 0.  Scores, mixing, sigmoids and sums are fp32, exp is the accurate expf; the result does not depend on
// how the prompt was cut into steps or on what else is in the batch.
//
//   sigmoid_attn_rows   one workgroup of four waves per (row, run of keys, block of outputs).  Per tile of 64 keys:
//                       A  lane = key: four query heads of one kv head at a time against the key row (read once from
//                          the cache), scores to LDS;
//                       B  lane = key, wave = heads w, w + 4, ..: mixing (talk rows are wave-uniform loads), sigmoid,
//                          weights to LDS;
//                       C  thread = (four heads of a kv head, one 16-byte chunk of the value, a share of the keys):
//                          weighted sums in registers, coalesced value rows.
//                       The shares are added in LDS, the runs of a row by a second launch.
//   kv_rows             k | v columns of a projection row into the pages, as they are
//   sigmoid_mfma        prompt portions on MFMA: sigmoid_prefill.hip
#include "../common.h"

using namespace dgi;

namespace {

template <typename T> __device__ __forceinline__ float ldf(const T* p);
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldf<uint16_t>(const uint16_t* p) { return bf16_to_f32(*p); }
template <typename T> __device__ __forceinline__ void stf(T* p, float v);
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void stf<uint16_t>(uint16_t* p, float v) { *p = f32_to_bf16(v); }

// E consecutive elements as floats: one 16-byte access (E = 16 / sizeof(T)) or a single element (E = 1)
template <typename T, int E> __device__ __forceinline__ void ldv(const T* p, float* f) {
  if constexpr (E == 1) {
    f[0] = ldf<T>(p);
  } else if constexpr (sizeof(T) == 2) {
    unpack8(*reinterpret_cast<const u32x4*>(p), f);
  } else {
    const float4 v = *reinterpret_cast<const float4*>(p);
    f[0] = v.x; f[1] = v.y; f[2] = v.z; f[3] = v.w;
  }
}

constexpr int NT = 256;
constexpr int RC = 4;          // query heads of one kv head handled together
constexpr int SP = 65;         // padded row of 64 keys in LDS

struct RowsArgs {
  const void *q, *k, *v;
  int q_stride;
  const int *block_tables, *cu_seqlens, *positions;
  int bt_stride, n_seqs, H, G, dk, dv, bs;
  float scale;
  int window;
  const float *talk, *pb;
  void* out;
  int out_stride, nsplit, rows;
  float* part;
};

// E: elements per access in the key / value rows
template <typename T, int E>
__global__ __launch_bounds__(NT) void sigmoid_attn_rows_kernel(const RowsArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int row = blockIdx.x, split = blockIdx.y;
  const int H = a.H, G = a.G, dk = a.dk, dv = a.dv, bs = a.bs;
  const int R = H / G, nrc = (R + RC - 1) / RC;
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63;
  float* qs = sm;                                        // [H][dk]
  float* ss = qs + ((H * dk + 3) & ~3);                  // [H][SP] raw scores, later the shares' sums [NT][RC * E]
  float* ws = ss + H * SP;                               // [H][SP] weights
  int* vs = reinterpret_cast<int*>(ws + H * SP);         // [64] cache slot of every key of the tile

  int seq = row;
  if (a.cu_seqlens) {
    int lo = 0, hi = a.n_seqs - 1;
    while (lo < hi) {
      const int mid = (lo + hi + 1) >> 1;
      if (a.cu_seqlens[mid] <= row) lo = mid; else hi = mid - 1;
    }
    seq = lo;
  }
  const int* bt = a.block_tables + (size_t)seq * a.bt_stride;
  const int pos = a.positions[row];
  const int first = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  const int tiles = (pos - first + 64) / 64;             // of 64 keys
  const int per = (tiles + a.nsplit - 1) / a.nsplit;
  const int k_lo = first + split * per * 64;
  const int k_hi = min(pos + 1, k_lo + per * 64);

  const T* qp = (const T*)a.q + (size_t)row * a.q_stride;
  for (int e = tid; e < H * dk; e += NT) qs[e] = ldf<T>(qp + e);

  // this thread's outputs: unit = (kv head, block of RC heads, chunk), and its share of a tile's keys
  const int nch = dv / E;
  const int nu = G * nrc * nch;
  const int u0 = blockIdx.z * NT;
  const int nub = min(NT, nu - u0);                      // units of this workgroup
  const int shares = NT / nub;
  const int ul = tid % nub, share = tid / nub;
  const int unit = u0 + ul;
  const int ch = unit % nch, rcb = (unit / nch) % nrc, ukv = unit / (nch * nrc);
  const int uh0 = ukv * R + rcb * RC;                    // first head
  const int unh = min(RC, R - rcb * RC);                 // heads of the unit
  float acc[RC][E];
#pragma unroll
  for (int i = 0; i < RC; ++i)
#pragma unroll
    for (int j = 0; j < E; ++j) acc[i][j] = 0.f;

  for (int k0 = k_lo; k0 < k_hi; k0 += 64) {
    const int n = min(64, k_hi - k0);
    const bool ok = lane < n;
    const int key = k0 + (ok ? lane : 0);
    const int blk = bt[key / bs], off = key % bs;
    __syncthreads();                                     // queries staged / the previous tile's weights read
    if (w == 0) vs[lane] = blk * G * bs + off;           // slot of kv head 0; kv head g adds g * bs
    for (int t = w; t < G * nrc; t += NT / 64) {
      const int kv = t / nrc, h0 = kv * R + (t % nrc) * RC, nh = min(RC, R - (t % nrc) * RC);
      const T* kp = (const T*)a.k + ((size_t)(blk * G + kv) * bs + off) * dk;
      const float* q0 = qs + h0 * dk;
      const float* q1 = nh > 1 ? q0 + dk : q0;
      const float* q2 = nh > 2 ? q1 + dk : q0;
      const float* q3 = nh > 3 ? q2 + dk : q0;
      float s0 = 0.f, s1 = 0.f, s2 = 0.f, s3 = 0.f;
#pragma unroll 2
      for (int e = 0; e < dk; e += E) {
        float kf[E];
        ldv<T, E>(kp + e, kf);
#pragma unroll
        for (int j = 0; j < E; ++j) {
          s0 += q0[e + j] * kf[j];
          s1 += q1[e + j] * kf[j];
          s2 += q2[e + j] * kf[j];
          s3 += q3[e + j] * kf[j];
        }
      }
      ss[h0 * SP + lane] = s0;
      if (nh > 1) ss[(h0 + 1) * SP + lane] = s1;
      if (nh > 2) ss[(h0 + 2) * SP + lane] = s2;
      if (nh > 3) ss[(h0 + 3) * SP + lane] = s3;
    }
    __syncthreads();
    for (int h = w; h < H; h += NT / 64) {
      float m = 0.f;
      if (a.talk) {
        const float* tr = a.talk + (size_t)h * H;
        for (int g = 0; g < H; ++g) m += tr[g] * ss[g * SP + lane];
      } else {
        m = ss[h * SP + lane];
      }
      m = m * a.scale + (a.pb ? a.pb[h] : 0.f);
      ws[h * SP + lane] = ok ? 1.f / (1.f + expf(-m)) : 0.f;
    }
    __syncthreads();
    if (share < shares) {
      const float* wp = ws + uh0 * SP;
      for (int kk = share; kk < n; kk += shares) {
        float vf[E];
        ldv<T, E>((const T*)a.v + (size_t)(vs[kk] + ukv * bs) * dv + ch * E, vf);
#pragma unroll
        for (int i = 0; i < RC; ++i) {
          const float p = i < unh ? wp[i * SP + kk] : 0.f;
#pragma unroll
          for (int j = 0; j < E; ++j) acc[i][j] += p * vf[j];
        }
      }
    }
  }
  // add the shares of a unit (share 0 stores); the reduction reuses the score / weight rows
  if (shares > 1) {
    float* red = ss;
#pragma unroll
    for (int i = 0; i < RC; ++i) {
      __syncthreads();
      if (share > 0 && share < shares) {
#pragma unroll
        for (int j = 0; j < E; ++j) red[(size_t)((share - 1) * nub + ul) * E + j] = acc[i][j];
      }
      __syncthreads();
      if (share == 0) {
        for (int s = 1; s < shares; ++s)
#pragma unroll
          for (int j = 0; j < E; ++j) acc[i][j] += red[(size_t)((s - 1) * nub + ul) * E + j];
      }
    }
  }
  if (share > 0) return;
#pragma unroll
  for (int i = 0; i < RC; ++i) {
    if (i >= unh) continue;
    const size_t c = (size_t)(uh0 + i) * dv + ch * E;
    if (a.nsplit > 1) {
      float* pp = a.part + ((size_t)split * a.rows + row) * H * dv + c;
#pragma unroll
      for (int j = 0; j < E; ++j) pp[j] = acc[i][j];
    } else {
      T* op = (T*)a.out + (size_t)row * a.out_stride + c;
#pragma unroll
      for (int j = 0; j < E; ++j) stf<T>(op + j, acc[i][j]);
    }
  }
}

// out[row] = sum of the row's runs, in their order
template <typename T>
__global__ __launch_bounds__(NT) void sigmoid_attn_sum_kernel(T* __restrict__ out, int out_stride, const float* __restrict__ part,
                                                              int nsplit, int rows, int C) {
  const int row = blockIdx.x;
  for (int c = blockIdx.y * NT + threadIdx.x; c < C; c += gridDim.y * NT) {
    float s = 0.f;
    for (int i = 0; i < nsplit; ++i) s += part[((size_t)i * rows + row) * C + c];
    stf<T>(out + (size_t)row * out_stride + c, s);
  }
}

template <typename T, int E>
__global__ __launch_bounds__(NT) void kv_rows_kernel(const T* __restrict__ kv, int stride, const int* __restrict__ slots, int T_,
                                                     int G, int dk, int dv, int bs, T* __restrict__ k_cache,
                                                     T* __restrict__ v_cache) {
  const int nk = G * dk / E, n = nk + G * dv / E;
  const long long total = (long long)T_ * n;
  for (long long i = (long long)blockIdx.x * NT + threadIdx.x; i < total; i += (long long)gridDim.x * NT) {
    const int t = (int)(i / n), u = (int)(i - (long long)t * n);
    const int slot = slots[t];
    if (slot < 0) continue;
    const int blk = slot / bs, off = slot - blk * bs;
    const bool isk = u < nk;
    const int e = (isk ? u : u - nk) * E, d = isk ? dk : dv;
    const int g = e / d, c = e - g * d;
    const T* src = kv + (size_t)t * stride + (isk ? 0 : G * dk) + e;
    T* dst = (isk ? k_cache : v_cache) + ((size_t)(blk * G + g) * bs + off) * d + c;
    if constexpr (E == 1) *dst = *src;
    else *reinterpret_cast<u32x4*>(dst) = *reinterpret_cast<const u32x4*>(src);
  }
}

template <typename T>
int launch_rows(const RowsArgs& a, bool vec, hipStream_t s) {
  constexpr int EV = 16 / sizeof(T);
  const int E = vec ? EV : 1;
  const int nu = a.G * ((a.H / a.G + RC - 1) / RC) * (a.dv / E);
  // score and weight rows are reused by the reduction of the shares: at most (NT - units) * E floats
  size_t score = (size_t)a.H * SP;
  const size_t red = (size_t)NT * E;
  size_t lds = ((size_t)((a.H * a.dk + 3) & ~3) + 2 * score + 64) * 4;
  if (2 * score + 64 < red) lds += (red - 2 * score - 64) * 4;
  if (lds > 160 * 1024) return -6;
  const dim3 grid(a.rows, a.nsplit, (nu + NT - 1) / NT);
  if (grid.y > 65535 || grid.z > 65535) return -7;
  const void* f = vec ? (const void*)sigmoid_attn_rows_kernel<T, EV> : (const void*)sigmoid_attn_rows_kernel<T, 1>;
  if (lds > 64 * 1024) {
    const hipError_t e = hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return (int)e;
  }
  if (vec) sigmoid_attn_rows_kernel<T, EV><<<grid, NT, lds, s>>>(a);
  else sigmoid_attn_rows_kernel<T, 1><<<grid, NT, lds, s>>>(a);
  DGI_CHECK_LAUNCH();
  if (a.nsplit > 1) {
    const int C = a.H * a.dv;
    const int gy = (C + NT - 1) / NT;
    sigmoid_attn_sum_kernel<T><<<dim3(a.rows, gy > 64 ? 64 : gy), NT, 0, s>>>((T*)a.out, a.out_stride, a.part, a.nsplit, a.rows, C);
    DGI_CHECK_LAUNCH();
  }
  return 0;
}

}  // namespace

// nsplit > 1: the keys of a row are cut into that many runs; part: [nsplit, rows, H * dv] fp32 scratch
extern "C" int dgi_sigmoid_attn_rows(const void* q, int q_stride, const void* k_cache, const void* v_cache,
                                     const int* block_tables, int bt_stride, const int* cu_seqlens, int n_seqs,
                                     const int* positions, int rows, int H, int G, int dk, int dv, int block_size, float scale,
                                     int window, const float* talk, const float* pb, void* out, int out_stride, int is_f32,
                                     int nsplit, float* part, hipStream_t s) {
  if (rows == 0) return 0;
  if (G <= 0 || H <= 0 || H % G || dk <= 0 || dv <= 0) return -2;
  if (window < 0 || nsplit < 1 || (nsplit > 1 && !part)) return -4;
  RowsArgs a;
  a.q = q; a.k = k_cache; a.v = v_cache; a.q_stride = q_stride;
  a.block_tables = block_tables; a.cu_seqlens = cu_seqlens; a.positions = positions;
  a.bt_stride = bt_stride; a.n_seqs = n_seqs; a.H = H; a.G = G; a.dk = dk; a.dv = dv; a.bs = block_size;
  a.scale = scale; a.window = window; a.talk = talk; a.pb = pb;
  a.out = out; a.out_stride = out_stride; a.nsplit = nsplit; a.rows = rows; a.part = part;
  const int E = is_f32 ? 4 : 8;
  const bool vec = dk % E == 0 && dv % E == 0 && ((uintptr_t)k_cache | (uintptr_t)v_cache) % 16 == 0;
  return is_f32 ? launch_rows<float>(a, vec, s) : launch_rows<uint16_t>(a, vec, s);
}

// kv: rows [k: G * dk | v: G * dv | ...] with their own stride; slots: page slot of every row (-1: not written)
extern "C" int dgi_kv_rows(const void* kv, int stride, const int* slots, int T, int G, int dk, int dv, int block_size,
                           void* k_cache, void* v_cache, int is_f32, hipStream_t s) {
  if (T == 0) return 0;
  if (G <= 0 || dk <= 0 || dv <= 0) return -2;
  const int E = is_f32 ? 4 : 8;
  const bool vec = dk % E == 0 && dv % E == 0 && stride % E == 0 &&
                   (((uintptr_t)kv | (uintptr_t)k_cache | (uintptr_t)v_cache) & 15) == 0;
  const long long n = (long long)T * (G * (dk + dv) / (vec ? E : 1));
  const unsigned blocks = (unsigned)((n + NT - 1) / NT > 65535 ? 65535 : (n + NT - 1) / NT);
#define DGI_KVR(TT_, EE_)                                                                                              \
  kv_rows_kernel<TT_, EE_><<<blocks, NT, 0, s>>>((const TT_*)kv, stride, slots, T, G, dk, dv, block_size, (TT_*)k_cache, \
                                                 (TT_*)v_cache)
  if (is_f32) { if (vec) DGI_KVR(float, 4); else DGI_KVR(float, 1); }
  else { if (vec) DGI_KVR(uint16_t, 8); else DGI_KVR(uint16_t, 1); }
#undef DGI_KVR
  DGI_CHECK_LAUNCH();
  return 0;
}
