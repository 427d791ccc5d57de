// dgi/csrc/mix/sigmoid_prefill.hip — prompt portions of sigmoid attention with mixed heads on MFMA (bf16; the definition is
// in sigmoid_attention.hip).  Mixing needs the scores of ALL heads of a (query, key) pair at once, so a workgroup
// owns 16 queries with all their heads and walks the visible keys in tiles of 32:
//
//   A  scores   wave = HW heads.  S^T = K Q^T, 16 keys x 16 queries per v_mfma_f32_16x16x32_bf16; the query fragments stay in
//               registers, key fragments come straight from the cache (each is used by one wave only; the heads of a
//               kv head share it).  fp32 scores go to LDS [head][query][key].
//   B  weights  wave = two queries, lane = (query, key).  A lane reads its pair's score of every head and mixes them with
//               v_mfma_f32_4x4x1_16b_f32: sixteen independent 4 x 4 products per instruction, i.e. every lane multiplies
//               its own score by four entries of the mixing matrix (broadcast from one register, cbsz / abid), fp32 all
//               the way and no data exchanged between lanes.  scale and log2(e) are folded into the matrix, the
//               number per head is one more product with a score of 1, so the weight is rcp(1 + exp2(acc)).  Weights
//               replace the scores in LDS as bf16 (the rows of a query belong to one wave).
//   C  values   wave = its heads again.  O^T += V^T P^T, one 16x16x32 product per 16 value dims; values were staged through
//               LDS by all waves (loads issued before B, stored after it) and are read transposed
//               (ds_read_b64_tr_b16).
//
// Heads beyond H (up to the padded count) have zero queries and zero rows / columns in the mixing matrix.
// More than 16 heads: a workgroup takes 8 queries, and the 16 columns of a product hold two heads of one kv head (QT == 8);
// the queries of a pair of waves are mixed by both, each for half of the output heads, so weights have rows of their
// own.  Where heads cannot be paired (an odd number of heads per kv head) the 16-query form runs, short of registers.
// Three barriers per tile.  Value rows in LDS are not padded; sizes of 64 and 128 swizzle their 16-byte chunks by row so that
// the four rows of a transposed read hit different banks.
// grid = 8 * (128-row query tiles); consecutive 16-row tiles go to one XCD (shared keys in its L2).
#include "../common.h"

using namespace dgi;

namespace {

constexpr int NW = 8;           // waves
constexpr int KT = 32;          // keys per tile
constexpr int SROW = 36;        // floats per (head, query) row of scores: 32 keys + padding
constexpr int PROW = 40;        // bf16 per row of weights where they do not replace the scores
constexpr int NVMAX = 8;        // value chunks staged per thread and tile, at most

struct PrefillArgs {
  const uint16_t *q, *k, *v;
  int q_stride;
  const int *block_tables, *cu, *ctx, *tiles;
  int bt_stride, H, G, dk, dv, bs_log2;
  float scale;
  int window;
  const float *talk, *pb;
  uint16_t* out;
  int out_stride;
};

// HP: heads padded to 4, 8, 16 or 32; NKS: 32-dim steps of a key; SHARE: the heads of a wave read one kv head; QT: queries;
// NVP: value chunks staged per thread and tile.  The tile loop has no branches: loads beyond a head's size or the last kv
// head repeat a valid address (their products are with zero, or never stored), so that waits stay exact.
template <int HP, int NKS, bool SHARE, int QT, int NVP>
__global__ __launch_bounds__(NW * 64, 2) void sigmoid_prefill_kernel(const PrefillArgs a) {
  constexpr int NWH = HP < NW ? HP : NW;          // groups of waves by head
  constexpr int NSP = NW / NWH;                   // waves per group: they split the keys (A) and the value dims (C)
  constexpr int HW = HP / NWH;                    // heads per wave
  constexpr int UH = 16 / QT;                     // heads per unit: a unit is the 16 columns of a product
  constexpr int HU = HW / UH;                     // units per wave
  constexpr bool PAIR = UH == 2;
  constexpr int NSUB = NSP >= 2 ? 1 : 2;          // 16-key halves of a tile per wave
  constexpr int NKV = SHARE ? 1 : HU;
  constexpr int NDT = 8 / NSP;                    // 16-dim value tiles per head and wave (value size at most 128)
  constexpr int HM = HP / 4;                      // groups of four mixed heads
  constexpr int TG = (HP + 15) / 16;              // registers per group of four rows of the mixing matrix
  constexpr int MW = PAIR ? HM / 2 : HM;          // groups mixed by one wave
  constexpr bool TLDS = MW > 4;                   // the matrix sits in LDS (registers are short)
  constexpr int MB = MW > 4 ? 4 : MW;             // groups mixed in one sweep over the scores
  static_assert(QT == 16 || (QT == 8 && HP == 32), "two heads per unit need four heads per wave");
  extern __shared__ __attribute__((aligned(16))) char lds[];
  float* S = reinterpret_cast<float*>(lds);       // [HP][QT][SROW]; weights: bf16 at the start of the same rows
  float* TM = S + HP * QT * SROW;                 // TLDS: [HM * TG][64]
  uint16_t* P = PAIR ? reinterpret_cast<uint16_t*>(TM) : reinterpret_cast<uint16_t*>(S);      // weights: rows of PS bf16
  constexpr int PS = PAIR ? PROW : 2 * SROW;
  uint16_t* V = reinterpret_cast<uint16_t*>(TM + (PAIR ? HP * QT * PROW / 2 : (TLDS ? HM * TG * 64 : 0)));      // [G][KT][dv]

  // QT-row tile of this workgroup: neighbours on one XCD (block b runs on XCD b % 8)
  constexpr int TPB = 128 / QT;
  const int per = gridDim.x >> 3;
  const int sub_tile = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
  const int b = a.tiles[2 * (sub_tile / TPB)];
  const int t0 = a.tiles[2 * (sub_tile / TPB) + 1] + QT * (sub_tile % TPB);
  const int q0 = a.cu[b];
  const int qlen = a.cu[b + 1] - q0;
  if (t0 >= qlen) return;
  const int ctx = a.ctx[b];
  const int pos0 = ctx - qlen + t0;               // position of the tile's first query
  const int last = min(t0 + QT, qlen) - 1 - t0;   // last query of the tile
  const int* bt = a.block_tables + (size_t)b * a.bt_stride;
  const int H = a.H, G = a.G, dk = a.dk, dv = a.dv, bs_log2 = a.bs_log2, bs = 1 << bs_log2;
  const int tid = threadIdx.x, w = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63;
  const int n16 = lane & 15, g16 = lane >> 4;
  const int R = H / G;
  const int hw0 = (w % NWH) * HW;                 // this wave's heads
  const int sp = w / NWH;
  const int uq = PAIR ? n16 & 7 : n16;            // query of this lane's column
  const int uh = PAIR ? n16 >> 3 : 0;             // head of this lane's column inside the unit

  // query fragments: lane = column n16, dims 32 s + 8 g16 ..
  u32x4 qf[HU][NKS];
#pragma unroll
  for (int i = 0; i < HU; ++i)
#pragma unroll
    for (int s = 0; s < NKS; ++s) {
      const int d = 32 * s + 8 * g16;
      const int h = hw0 + UH * i + uh;
      const bool ok = h < H && uq <= last && d < dk;
      qf[i][s] = ok ? *reinterpret_cast<const u32x4*>(a.q + (size_t)(q0 + t0 + uq) * a.q_stride + h * dk + d)
                    : u32x4{0, 0, 0, 0};
    }
  // mixing matrix: register (m, t) lane l holds T[4 m + l % 4][16 t + l / 4], times -scale log2(e)
  const float neg = -1.4426950408889634f;
  float tm[TLDS ? 1 : MW][TG], pbm[MW];
  const int mbase = PAIR ? (w >> 2) * MW : 0;      // first group of four output heads this wave mixes
#pragma unroll
  for (int m = 0; m < MW; ++m) {
    const int r = 4 * (mbase + m) + (lane & 3);
    pbm[m] = (a.pb && r < H) ? a.pb[r] * neg : 0.f;
#pragma unroll
    for (int t = 0; t < TG; ++t) {
      const int c = 16 * t + (lane >> 2);
      float x = (r < H && c < H) ? (a.talk ? a.talk[r * H + c] : (r == c ? 1.f : 0.f)) : 0.f;
      x *= a.scale * neg;
      if constexpr (TLDS) {
        if (w == 0) TM[(m * TG + t) * 64 + lane] = x;
      } else {
        tm[m][t] = x;
      }
    }
  }
  f32x4 o[HU][NDT];
#pragma unroll
  for (int i = 0; i < HU; ++i)
#pragma unroll
    for (int d = 0; d < NDT; ++d) o[i][d] = f32x4{0.f, 0.f, 0.f, 0.f};

  const int kv_lo = a.window > 0 ? max(0, pos0 - a.window + 1) : 0;
  const int kv_hi = pos0 + last + 1;              // one past the last visible key (at most ctx)
  const int mq = 2 * (PAIR ? w & 3 : w) + (lane >> 5), mk = lane & 31;      // phase B: this lane's query and key
  const int mpos = pos0 + mq;
  const int mfirst = a.window > 0 ? max(0, mpos - a.window + 1) : 0;

  // value staging: 2^cl lanes per row, a thread keeps its key and chunk and steps over the kv heads
  const int chv = dv >> 3;                        // 16-byte chunks per value row
  const int cl = chv <= 4 ? 2 : (chv <= 8 ? 3 : 4);
  const int vk = (tid >> cl) & (KT - 1), vc = tid & ((1 << cl) - 1), vg0 = tid >> (cl + 5), vgs = 16 >> cl;
  auto swz = [&](int row) { return dv == 128 ? (row & 3) << 2 : (dv == 64 ? ((row >> 1) & 1) << 2 : 0); };
  // cache slot (kv head 0) of key kb + lane % 32; kv head g is g << bs_log2 further
  const int vcc = min(vc, chv - 1);
  uint16_t* vdst = V + vk * dv + (vcc ^ swz(vk)) * 8;
  int kd[NKS];                                    // this lane's dims of a key row
#pragma unroll
  for (int s = 0; s < NKS; ++s) kd[s] = min(32 * s + 8 * g16, dk - 8);
  // (its page is looked up a tile ahead and kept as loaded: arithmetic on it would wait for the load on the spot)
  auto page_of = [&](int kb) { return bt[min(kb + mk, kv_hi - 1) >> bs_log2]; };
  auto slot_of = [&](int page, int kb) { return ((page * G) << bs_log2) + (min(kb + mk, kv_hi - 1) & (bs - 1)); };
  u32x4 kf[NSUB][NKV][NKS];
  auto load_k = [&](int slot, int j) {           // 16-key half j of the wave's keys
    {
      const int kk = 16 * (NSUB == 1 ? (sp & 1) : j) + n16;
      const int sl = __shfl(slot, kk, 64);
#pragma unroll
      for (int i = 0; i < NKV; ++i) {
        const int h = min(hw0 + UH * i, H - 1);
        const uint16_t* kp = a.k + ((size_t)sl + ((size_t)(h / R) << bs_log2)) * dk;
#pragma unroll
        for (int s = 0; s < NKS; ++s) kf[j][i][s] = *reinterpret_cast<const u32x4*>(kp + kd[s]);
      }
    }
  };
  int page = page_of(kv_lo), page1 = page_of(kv_lo + KT);      // of the tile, of the next one
  u32x4 vr[NVP];
  auto load_v = [&](int slot) {
    const int sl = __shfl(slot, vk, 64);
#pragma unroll
    for (int p = 0; p < NVP; ++p) {
      const int g = min(vg0 + p * vgs, G - 1);
      vr[p] = *reinterpret_cast<const u32x4*>(a.v + ((size_t)sl + ((size_t)g << bs_log2)) * dv + vcc * 8);
    }
  };
#pragma unroll
  for (int j = 0; j < NSUB; ++j) load_k(slot_of(page, kv_lo), j);
  load_v(slot_of(page, kv_lo));

  for (int kb = kv_lo; kb < kv_hi; kb += KT) {
    // ---- A: scores of this wave's heads
    {
#pragma unroll
      for (int j = 0; j < NSUB; ++j) {
        const int ks = 16 * (NSUB == 1 ? (sp & 1) : j);
#pragma unroll
        for (int i = 0; i < HU; ++i) {
          f32x4 sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int s = 0; s < NKS; ++s)
            sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(kf[j][SHARE ? 0 : i][s]), as_bf16x8(qf[i][s]), sc, 0, 0, 0);
          *reinterpret_cast<f32x4*>(S + ((hw0 + UH * i + uh) * QT + uq) * SROW + ks + 4 * g16) = sc;
        }
      }
    }
    __syncthreads();

    // ---- B: mix the heads of one (query, key) pair per lane, weights back to LDS
    {
      // keys of the next tile, spread over the mixing: a wave that issues all its loads at once waits for the
      // address unit instead of computing
      page = page1;
      page1 = page_of(kb + 2 * KT);
      const int slot1 = slot_of(page, kb + KT);
      const int key = kb + mk;
      const bool ok = mq <= last && key <= mpos && key >= mfirst;
      const float* sr = S + mq * SROW + mk;
      uint32_t pk[MW][2];                          // weights of four heads as bf16
#pragma unroll
      for (int m0 = 0; m0 < MW; m0 += MB) {
        f32x4 acc[MB];
#pragma unroll
        for (int m = 0; m < MB; ++m)
          acc[m] = __builtin_amdgcn_mfma_f32_4x4x1f32(pbm[m0 + m], 1.f, f32x4{0.f, 0.f, 0.f, 0.f}, 0, 0, 0);
        float tl[TLDS ? MB : 1][TG];
        if constexpr (TLDS) {
#pragma unroll
          for (int m = 0; m < MB; ++m)
#pragma unroll
            for (int t = 0; t < TG; ++t) tl[m][t] = TM[((m0 + m) * TG + t) * 64 + lane];
        }
#define DGI_MIX(G_)                                                                                        \
        if constexpr (G_ < HP) {                                                                           \
          const float sv = sr[(G_) * QT * SROW];                                                           \
          _Pragma("unroll") for (int m = 0; m < MB; ++m) {                                                 \
            float tv;                                                                                      \
            if constexpr (TLDS) tv = tl[m][(G_) / 16];                                                     \
            else tv = tm[m0 + m][(G_) / 16];                                                               \
            acc[m] = __builtin_amdgcn_mfma_f32_4x4x1f32(tv, sv, acc[m], 4, (G_) & 15, 0);                  \
          }                                                                                                \
        }
        if (m0 == 0) load_k(slot1, 0);
        __builtin_amdgcn_sched_barrier(0);
        DGI_MIX(0) DGI_MIX(1) DGI_MIX(2) DGI_MIX(3) DGI_MIX(4) DGI_MIX(5) DGI_MIX(6) DGI_MIX(7)
        __builtin_amdgcn_sched_barrier(0);
        if (NSUB > 1 && m0 == 0) load_k(slot1, NSUB - 1);
        __builtin_amdgcn_sched_barrier(0);
        DGI_MIX(8) DGI_MIX(9) DGI_MIX(10) DGI_MIX(11) DGI_MIX(12) DGI_MIX(13) DGI_MIX(14) DGI_MIX(15)
        DGI_MIX(16) DGI_MIX(17) DGI_MIX(18) DGI_MIX(19) DGI_MIX(20) DGI_MIX(21) DGI_MIX(22) DGI_MIX(23)
        DGI_MIX(24) DGI_MIX(25) DGI_MIX(26) DGI_MIX(27) DGI_MIX(28) DGI_MIX(29) DGI_MIX(30) DGI_MIX(31)
#undef DGI_MIX
#pragma unroll
        for (int m = 0; m < MB; ++m) {
          float p[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) p[r] = ok ? __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(acc[m][r])) : 0.f;
          pk[m0 + m][0] = pack_bf16x2(p[0], p[1]);
          pk[m0 + m][1] = pack_bf16x2(p[2], p[3]);
        }
      }
      asm volatile("" ::: "memory");               // every score of the pair is read before a weight overwrites the row
      uint16_t* pr = P + (4 * mbase * QT + mq) * PS + mk;
#pragma unroll
      for (int m = 0; m < MW; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          pr[(4 * m + r) * QT * PS] = (uint16_t)((r & 1) ? pk[m][r >> 1] >> 16 : pk[m][r >> 1] & 0xffffu);
      asm volatile("" ::: "memory");
    }
#pragma unroll
    for (int p = 0; p < NVP; ++p) *reinterpret_cast<u32x4*>(vdst + min(vg0 + p * vgs, G - 1) * (KT * dv)) = vr[p];
    __syncthreads();

    // ---- C: values (those of the next tile are loaded meanwhile)
    {
      load_v(slot_of(page, kb + KT));
      __builtin_amdgcn_sched_barrier(0);
      const int tq = n16 >> 2, tp = n16 & 3;
      u32x4 pf[HU];
#pragma unroll
      for (int i = 0; i < HU; ++i)
        pf[i] = *reinterpret_cast<const u32x4*>(P + ((hw0 + UH * i + uh) * QT + uq) * PS + 8 * g16);
      const uint16_t* vrow[NKV];
#pragma unroll
      for (int i = 0; i < NKV; ++i) vrow[i] = V + ((min(hw0 + UH * i, H - 1) / R) * KT + 8 * g16 + tq) * dv + 4 * tp;
      const int xv = swz(tq);                      // the same for rows 4 apart
#pragma unroll
      for (int d = 0; d < NDT; ++d) {
        const int c = ((2 * min(d * NSP + sp, (dv >> 4) - 1)) ^ xv) * 8;
        u32x4 vf;
#pragma unroll
        for (int i = 0; i < HU; ++i) {
          if (i == 0 || !SHARE) {
            const uint16_t* vp = vrow[SHARE ? 0 : i] + c;
            const short4v lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_short4*)vp);
            const short4v hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_short4*)(vp + 4 * dv));
            vf[0] = (uint32_t)(uint16_t)lo[0] | ((uint32_t)(uint16_t)lo[1] << 16);
            vf[1] = (uint32_t)(uint16_t)lo[2] | ((uint32_t)(uint16_t)lo[3] << 16);
            vf[2] = (uint32_t)(uint16_t)hi[0] | ((uint32_t)(uint16_t)hi[1] << 16);
            vf[3] = (uint32_t)(uint16_t)hi[2] | ((uint32_t)(uint16_t)hi[3] << 16);
          }
          o[i][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(vf), as_bf16x8(pf[i]), o[i][d], 0, 0, 0);
        }
      }
    }
    __syncthreads();                               // weights and values are consumed
  }

  if (uq > last) return;
#pragma unroll
  for (int i = 0; i < HU; ++i) {
    const int h = hw0 + UH * i + uh;
    if (h >= H) continue;
    uint16_t* op = a.out + (size_t)(q0 + t0 + uq) * a.out_stride + (size_t)h * dv;
#pragma unroll
    for (int d = 0; d < NDT; ++d) {
      const int dt = d * NSP + sp;
      if (16 * dt < dv) {
        uint2 r;
        r.x = pack_bf16x2(o[i][d][0], o[i][d][1]);
        r.y = pack_bf16x2(o[i][d][2], o[i][d][3]);
        *reinterpret_cast<uint2*>(op + 16 * dt + 4 * g16) = r;
      }
    }
  }
}

int padded_heads(int H) { return H <= 4 ? 4 : (H <= 8 ? 8 : (H <= 16 ? 16 : (H <= 32 ? 32 : 0))); }
// queries per workgroup
int query_tile(int HP, int R) { return HP == 32 && R % 2 == 0 ? 8 : 16; }
size_t lds_bytes(int HP, int R, int G, int dv) {
  const int QT = query_tile(HP, R);
  const size_t extra = QT == 8 ? (size_t)HP * QT * PROW * 2 : (HP > 16 ? (size_t)(HP / 4) * ((HP + 15) / 16) * 256 : 0);
  return (size_t)HP * QT * SROW * 4 + extra + (size_t)G * KT * dv * 2;
}

template <int HP, int NKS, bool SHARE, int QT, int NVP>
int launch_one(const PrefillArgs& a, int n_tiles, size_t lds, hipStream_t s) {
  auto kernel = sigmoid_prefill_kernel<HP, NKS, SHARE, QT, NVP>;
  if (lds > 64 * 1024) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return (int)e;
  }
  kernel<<<n_tiles * (128 / QT), NW * 64, lds, s>>>(a);
  return 0;
}

// kv heads one staging pass covers
int kv_per_pass(int dv) { return dv <= 32 ? 4 : (dv <= 64 ? 2 : 1); }

template <int HP, int NKS, bool SHARE, int QT>
int launch_passes(const PrefillArgs& a, int n_tiles, size_t lds, hipStream_t s) {
  const int passes = (a.G + kv_per_pass(a.dv) - 1) / kv_per_pass(a.dv);
  if (passes <= 2) return launch_one<HP, NKS, SHARE, QT, 2>(a, n_tiles, lds, s);
  if (passes <= 4) return launch_one<HP, NKS, SHARE, QT, 4>(a, n_tiles, lds, s);
  return launch_one<HP, NKS, SHARE, QT, NVMAX>(a, n_tiles, lds, s);
}

template <int HP, bool SHARE, int QT = 16>
int launch_dims(const PrefillArgs& a, int n_tiles, size_t lds, hipStream_t s) {
  if (a.dk <= 64) return launch_passes<HP, 2, SHARE, QT>(a, n_tiles, lds, s);
  return launch_passes<HP, 4, SHARE, QT>(a, n_tiles, lds, s);
}

}  // namespace

// whether the MFMA kernel serves this geometry (0 / 1); the row kernel serves every other
extern "C" int dgi_sigmoid_prefill_ok(int H, int G, int dk, int dv) {
  const int HP = padded_heads(H);
  return HP > 0 && G > 0 && H % G == 0 && dk % 8 == 0 && dk <= 128 && dv % 16 == 0 && dv <= 128 &&
         G <= NVMAX * kv_per_pass(dv) && lds_bytes(HP, H / G, G, dv) <= 160 * 1024;
}

// tiles: int32 [n_tiles, 2] = (sequence index, first query row of a 128-row tile)
extern "C" int dgi_sigmoid_prefill(const void* q, int q_stride, const void* k_cache, const void* v_cache, const int* block_tables,
                                   int bt_stride, const int* cu_seqlens_q, const int* context_lens, const int* tiles, int n_tiles,
                                   void* out, int out_stride, int H, int G, int dk, int dv, int block_size, float scale, int window,
                                   const float* talk, const float* pb, hipStream_t s) {
  if (n_tiles == 0) return 0;
  if (!dgi_sigmoid_prefill_ok(H, G, dk, dv) || window < 0) return -5;
  int bs_log2 = 0;
  while ((1 << bs_log2) < block_size) ++bs_log2;
  if ((1 << bs_log2) != block_size) return -4;
  PrefillArgs a;
  a.q = (const uint16_t*)q; a.k = (const uint16_t*)k_cache; a.v = (const uint16_t*)v_cache; a.q_stride = q_stride;
  a.block_tables = block_tables; a.cu = cu_seqlens_q; a.ctx = context_lens; a.tiles = tiles;
  a.bt_stride = bt_stride; a.H = H; a.G = G; a.dk = dk; a.dv = dv; a.bs_log2 = bs_log2;
  a.scale = scale; a.window = window; a.talk = talk; a.pb = pb;
  a.out = (uint16_t*)out; a.out_stride = out_stride;
  const int HP = padded_heads(H), HW = HP > NW ? HP / NW : 1, R = H / G;
  const bool share = R % HW == 0;                  // every wave's heads (HW consecutive ones) lie in one kv head
  const size_t lds = lds_bytes(HP, R, G, dv);
  int rc;
  if (HP == 4) rc = launch_dims<4, true>(a, n_tiles, lds, s);
  else if (HP == 8) rc = launch_dims<8, true>(a, n_tiles, lds, s);
  else if (HP == 16) rc = share ? launch_dims<16, true>(a, n_tiles, lds, s) : launch_dims<16, false>(a, n_tiles, lds, s);
  else if (query_tile(HP, R) == 8)
    rc = share ? launch_dims<32, true, 8>(a, n_tiles, lds, s) : launch_dims<32, false, 8>(a, n_tiles, lds, s);
  else
    rc = launch_dims<32, false>(a, n_tiles, lds, s);
  if (rc) return rc;
  DGI_CHECK_LAUNCH();
  return 0;
}
