// dgi/csrc/mix/moe_group.hip — routing and experts of a step on the matrix cores (bf16), without a host round trip.
//
//   moe_router   router logits and the choice in one launch: z = h R^T with R in bf16 (products of bf16 numbers are exact
//                in fp32 and are summed in fp32), then sigmoid scores, the `top` largest (ties: lowest index), optionally
//                divided by their sum, times a factor.  A workgroup owns 16 tokens, its waves share K.
//   moe_plan     sorts the step's (token, route) pairs by expert: order[place] = pair, where[pair] = place and
//                seg[e] .. seg[e + 1] = the places of expert e; pairs of identity routes (e >= E) get no place.  One
//                workgroup per expert reads all routes, counts those of smaller experts (its first place) and lists its
//                own in pair order, so the sort is stable and needs no scan across workgroups.
//   moe_group    out[place][n] = A[row(place)] . B[e][n], n < N, for every place of every expert, with
//                  gate-up (GLU): B = gate_up [E, 2 ff, K], A = the step's hidden rows, row(place) = order[place] / top, and
//                                 out [places, ff] = act(s g, s u), s = pair_scale[order[place]] (or 1): the two projections
//                                 of an output sit in the same lane, so the activation is the product's epilogue;
//                  down:          B = down [E, N, K], A = the rows gate-up left, row(place) = place.
//
// Two kernels.  Few rows per expert (decode steps): bounded by the expert weights' bytes.  A workgroup owns 64 weight
// rows and up to 64 places; its four waves take a quarter of K each, weights and rows go from memory straight into
// operand registers (16x16x32 products), and the four partial sums meet in LDS.  Many rows: tiles of 128 places by 128
// weight rows, K in steps of 64 through two LDS stages (32x32x16 products).
//
// The tile a workgroup owns is found from seg alone, so the grid is sized for the worst split of the places over the
// experts and a workgroup past the last tile leaves.  Weights are the A operand: a lane's result is four consecutive
// outputs of one place.  K must be a multiple of 8; N and the number of places are free.
#include "../common.h"

using namespace dgi;

namespace {

constexpr int PLAN_NT = 1024;

__global__ __launch_bounds__(PLAN_NT) void moe_plan_kernel(const int* __restrict__ idx, int P, int E, int* __restrict__ order,
                                                           int* __restrict__ where, int* __restrict__ seg) {
  __shared__ int red[2][PLAN_NT / 64];
  const int e = blockIdx.x, tid = threadIdx.x, w = tid >> 6, lane = tid & 63;
  int less = 0, mine = 0;
  for (int p = tid; p < P; p += PLAN_NT) {
    const int r = idx[p];
    less += (r >= 0 && r < e) ? 1 : 0;
    mine += r == e ? 1 : 0;
  }
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    less += __shfl_xor(less, o, 64);
    mine += __shfl_xor(mine, o, 64);
  }
  if (lane == 0) { red[0][w] = less; red[1][w] = mine; }
  __syncthreads();
  less = mine = 0;
#pragma unroll
  for (int i = 0; i < PLAN_NT / 64; ++i) { less += red[0][i]; mine += red[1][i]; }
  if (tid == 0) {
    seg[e] = less;
    if (e == E - 1) seg[E] = less + mine;
  }
  int at = less;                                       // next place of this expert
  for (int p0 = 0; p0 < P && mine > 0; p0 += PLAN_NT) {
    const int p = p0 + tid;
    const bool hit = p < P && idx[p] == e;
    const unsigned long long m = __ballot(hit);
    __syncthreads();                                   // red of the round before is read
    if (lane == 0) red[0][w] = __popcll(m);
    __syncthreads();
    int before = 0, all = 0;
#pragma unroll
    for (int i = 0; i < PLAN_NT / 64; ++i) {
      const int c = red[0][i];
      before += i < w ? c : 0;
      all += c;
    }
    if (hit) {
      const int place = at + before + __popcll(m & ((1ull << lane) - 1ull));
      order[place] = p;
      where[p] = place;
    }
    at += all;
  }
}

// The m-tile `tile` of BM places: its expert and places [lo, hi); false past the last tile.  Uniform over the wave.
template <int BM>
__device__ __forceinline__ bool find_tile(const int* __restrict__ seg, int E, int tile, int& e, int& lo, int& hi) {
  const int lane = threadIdx.x & 63;
  int base = 0;                                        // tiles of the experts before this round's 64
  for (int e0 = 0; e0 < E; e0 += 64) {
    const int ee = e0 + lane;
    const int s0 = ee < E ? seg[ee] : 0, s1 = ee < E ? seg[ee + 1] : 0;
    const int n = (s1 - s0 + BM - 1) / BM;
    int inc = n;                                       // inclusive prefix over the lanes
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int v = __shfl_up(inc, o, 64);
      if (lane >= o) inc += v;
    }
    const unsigned long long m = __ballot(base + inc > tile);
    if (m) {
      const int l = __ffsll(m) - 1;
      const int first = base + __shfl(inc - n, l, 64);
      e = e0 + l;
      lo = __shfl(s0, l, 64) + (tile - first) * BM;
      hi = min(__shfl(s1, l, 64), lo + BM);
      return true;
    }
    base += __shfl(inc, 63, 64);
  }
  return false;
}

// expert activation: kind 0 silu(g) * u; kind 1 the clamped sigmoid-GLU
__device__ __forceinline__ float glu_f(float g, float u, int kind, float limit, float alpha) {
  if (kind == 1) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g / (1.f + __expf(-alpha * g)) * (u + 1.f);
  }
  return g / (1.f + __expf(-g)) * u;
}

struct GroupArgs {
  const uint16_t* a;          // rows of K
  int a_stride;
  const uint16_t* b;          // [E, NB, K] (NB = N, or 2 N with the gate rows first)
  uint16_t* out;              // [places, N]
  const int* seg;
  const int* order;           // gate-up: place -> pair; down: nullptr (row = place)
  const float* pair_scale;    // gate-up: factor of g and u by pair, or nullptr
  int E, N, K, top, act;
  float limit, alpha;
  int mtiles;
};

__device__ __forceinline__ void st_out4(uint16_t* p, const float* v, int n, bool vec) {
  if (vec && n == 4) {
    *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i < n) p[i] = f32_to_bf16(v[i]);
  }
}

// ---- few rows per expert: MB blocks of 16 places, 64 weight rows (GLU: 32 outputs, gate and up), K over four waves
template <int MB, bool GLU>
__global__ __launch_bounds__(256) void moe_group_rows_kernel(GroupArgs g) {
  __shared__ __attribute__((aligned(16))) float part[4][MB * 4][64][4];
  const int w = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int lr = lane & 15, lg = lane >> 4;
  int e, lo, hi;
  if (!find_tile<16 * MB>(g.seg, g.E, blockIdx.x % g.mtiles, e, lo, hi)) return;
  const int nt = blockIdx.x / g.mtiles;
  constexpr int NO = GLU ? 32 : 64;                    // outputs per workgroup
  const int n0 = nt * NO;
  const uint16_t* B = g.b + (size_t)e * (GLU ? 2 : 1) * g.N * g.K;
  // this lane's weight rows: block j of 16 (GLU: two gate blocks, then the matching up blocks)
  const uint16_t* wp[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int n = n0 + (GLU ? (j & 1) : j) * 16 + lr;
    wp[j] = B + ((size_t)min(n, g.N - 1) + (GLU && j >= 2 ? g.N : 0)) * g.K;
  }
  const uint16_t* ap[MB];
#pragma unroll
  for (int i = 0; i < MB; ++i) {
    const int place = min(lo + 16 * i + lr, hi - 1);
    const int row = g.order ? g.order[place] / g.top : place;
    ap[i] = g.a + (size_t)row * g.a_stride;
  }
  f32x4 acc[MB][4];
#pragma unroll
  for (int i = 0; i < MB; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  // K in steps of 32; wave w takes a contiguous quarter of them.  U steps are loaded together.
  constexpr int U = MB == 1 ? 4 : 2;
  const int steps = (g.K + 31) >> 5, per = (steps + 3) >> 2;
  const int s_lo = w * per, s_hi = min(steps, s_lo + per);
  const u32x4 zero = {0u, 0u, 0u, 0u};
  for (int s = s_lo; s < s_hi; s += U) {
    u32x4 wf[U][4], af[U][MB];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = (s + u) * 32 + 8 * lg;
      const bool ok = s + u < s_hi && k < g.K;         // K is a multiple of 8: a chunk is whole or absent
#pragma unroll
      for (int j = 0; j < 4; ++j) wf[u][j] = ok ? *reinterpret_cast<const u32x4*>(wp[j] + k) : zero;
#pragma unroll
      for (int i = 0; i < MB; ++i) af[u][i] = ok ? *reinterpret_cast<const u32x4*>(ap[i] + k) : zero;
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int i = 0; i < MB; ++i)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(wf[u][j]), as_bf16x8(af[u][i]), acc[i][j], 0, 0, 0);
  }
#pragma unroll
  for (int i = 0; i < MB; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) *reinterpret_cast<f32x4*>(part[w][i * 4 + j][lane]) = acc[i][j];
  __syncthreads();
  auto total = [&](int blk) {
    f32x4 t = *reinterpret_cast<const f32x4*>(part[0][blk][lane]);
#pragma unroll
    for (int ww = 1; ww < 4; ++ww) {
      const f32x4 v = *reinterpret_cast<const f32x4*>(part[ww][blk][lane]);
#pragma unroll
      for (int r = 0; r < 4; ++r) t[r] += v[r];
    }
    return t;
  };
  constexpr int ITEMS = MB * (GLU ? 2 : 4);            // (block of places, block of 16 outputs)
  const bool vec = (g.N & 3) == 0 && ((uintptr_t)g.out & 7) == 0;
  for (int it = w; it < ITEMS; it += 4) {
    const int i = GLU ? it >> 1 : it >> 2, j = GLU ? it & 1 : it & 3;
    const int place = lo + 16 * i + lr, n = n0 + 16 * j + 4 * lg;
    const f32x4 x = total(i * 4 + j);
    float v[4];
    if constexpr (GLU) {
      const f32x4 y = total(i * 4 + 2 + j);
      const float ps = g.pair_scale && place < hi ? g.pair_scale[g.order[place]] : 1.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = glu_f(x[r] * ps, y[r] * ps, g.act, g.limit, g.alpha);
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = x[r];
    }
    if (place < hi && n < g.N) st_out4(g.out + (size_t)place * g.N + n, v, min(4, g.N - n), vec);
  }
}

// ---- many rows per expert: 128 places x 128 weight rows (GLU: 64 outputs, gate and up), 64 of K per LDS stage.
// LDS row of 64 elements = eight 16-byte chunks, chunk c of row r at c ^ (r & 7).
__device__ __forceinline__ int sw(int row, int c) { return row * 64 + ((c ^ (row & 7)) << 3); }

template <bool GLU>
__global__ __launch_bounds__(256, 2) void moe_group_tiles_kernel(GroupArgs g, int n_tiles) {
  __shared__ __attribute__((aligned(16))) uint16_t lds[2][2][128 * 64];       // [stage][rows | weights]
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63;
  const int lr = lane & 31, hh = lane >> 5;
  // consecutive workgroups go to different XCDs: give every XCD a contiguous run of tiles, all m-tiles of a weight tile
  // in a row, so its L2 sees each weight tile once
  const int total = g.mtiles * n_tiles, chunk = (total + 7) / 8;
  const int id = (blockIdx.x & 7) * chunk + (blockIdx.x >> 3);
  if (id >= total) return;
  int e, lo, hi;
  if (!find_tile<128>(g.seg, g.E, id % g.mtiles, e, lo, hi)) return;
  constexpr int NO = GLU ? 64 : 128;
  const int n0 = (id / g.mtiles) * NO;
  const uint16_t* B = g.b + (size_t)e * (GLU ? 2 : 1) * g.N * g.K;
  // staging: thread -> chunk c of rows r0 + 32 i
  const int c = tid & 7, r0 = tid >> 3;
  const uint16_t *ap[4], *bp[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = r0 + 32 * i;
    const int place = min(lo + r, hi - 1);
    ap[i] = g.a + (size_t)(g.order ? g.order[place] / g.top : place) * g.a_stride + c * 8;
    // GLU weight rows: wave column wn owns rows 64 wn .. of the stage: 32 gate rows, then the matching 32 up rows
    const int n = GLU ? n0 + 32 * (r >> 6) + (r & 31) : n0 + r;
    bp[i] = B + ((size_t)min(n, g.N - 1) + (GLU && (r & 32) ? g.N : 0)) * g.K + c * 8;
  }
  u32x4 ra[4], rb[4];
  const u32x4 zero = {0u, 0u, 0u, 0u};
  const int steps = (g.K + 63) >> 6;
  auto load = [&](int s) {
    const bool ok = s * 64 + c * 8 < g.K;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      ra[i] = ok ? *reinterpret_cast<const u32x4*>(ap[i] + s * 64) : zero;
      rb[i] = ok ? *reinterpret_cast<const u32x4*>(bp[i] + s * 64) : zero;
    }
  };
  auto store = [&](int st) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      *reinterpret_cast<u32x4*>(&lds[st][0][sw(r0 + 32 * i, c)]) = ra[i];
      *reinterpret_cast<u32x4*>(&lds[st][1][sw(r0 + 32 * i, c)]) = rb[i];
    }
  };
  const int wm = w >> 1, wn = w & 1;                   // 64 places x 64 weight rows per wave
  f32x16 acc[2][2];                                    // [places block][weights block]
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[i][j][r] = 0.f;
  load(0);
  store(0);
  if (steps > 1) load(1);
  __syncthreads();
  for (int s = 0; s < steps; ++s) {
    const uint16_t* as = lds[s & 1][0];
    const uint16_t* bs = lds[s & 1][1];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      u32x4 fa[2], fb[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        fa[i] = *reinterpret_cast<const u32x4*>(as + sw(64 * wm + 32 * i + lr, 2 * k + hh));
        fb[i] = *reinterpret_cast<const u32x4*>(bs + sw(64 * wn + 32 * i + lr, 2 * k + hh));
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(as_bf16x8(fb[j]), as_bf16x8(fa[i]), acc[i][j], 0, 0, 0);
    }
    if (s + 1 < steps) {
      store((s + 1) & 1);                              // the stage read in step s - 1: every wave is past that step's barrier
      if (s + 2 < steps) load(s + 2);
    }
    __syncthreads();
  }
  const bool vec = (g.N & 3) == 0 && ((uintptr_t)g.out & 7) == 0;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int place = lo + 64 * wm + 32 * i + lr;
    if (place >= hi) continue;
    uint16_t* orow = g.out + (size_t)place * g.N;
    const float ps = GLU && g.pair_scale ? g.pair_scale[g.order[place]] : 1.f;
#pragma unroll
    for (int j = 0; j < (GLU ? 1 : 2); ++j)
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int n = n0 + (GLU ? 32 * wn : 64 * wn + 32 * j) + 8 * q + 4 * hh;
        if (n >= g.N) continue;
        float v[4];
#pragma unroll
        for (int r = 0; r < 4; ++r)
          v[r] = GLU ? glu_f(acc[i][0][4 * q + r] * ps, acc[i][1][4 * q + r] * ps, g.act, g.limit, g.alpha) : acc[i][j][4 * q + r];
        st_out4(orow + n, v, min(4, g.N - n), vec);
      }
  }
}

template <bool GLU>
int launch_group(GroupArgs g, int places, int rows_per_tile, hipStream_t s) {
  // worst split of the places over the experts: every non-empty expert may end in a partial tile
  const int nonempty = g.E < places ? g.E : places;
  const int bm = rows_per_tile;
  g.mtiles = places / bm + nonempty;
  const int no = (bm == 128 ? 128 : 64) / (GLU ? 2 : 1);
  const int ntn = (g.N + no - 1) / no;
  const long long blocks = (long long)g.mtiles * ntn;
  if (blocks > 0x3fffffff) return -4;
  if (bm == 128) {
    const int padded = (int)((blocks + 7) / 8 * 8);
    moe_group_tiles_kernel<GLU><<<padded, 256, 0, s>>>(g, ntn);
  } else if (bm == 64) {
    moe_group_rows_kernel<4, GLU><<<(int)blocks, 256, 0, s>>>(g);
  } else if (bm == 32) {
    moe_group_rows_kernel<2, GLU><<<(int)blocks, 256, 0, s>>>(g);
  } else if (bm == 16) {
    moe_group_rows_kernel<1, GLU><<<(int)blocks, 256, 0, s>>>(g);
  } else {
    return -3;
  }
  return 0;
}

// EB blocks of 16 experts; NW waves split K; logits meet in LDS, then wave w routes tokens w, w + NW, ...
constexpr int RNW = 16;

template <int EB>
__global__ __launch_bounds__(64 * RNW) void moe_router_kernel(int* __restrict__ idx, float* __restrict__ wts,
                                                              const uint16_t* __restrict__ h, int h_stride,
                                                              const uint16_t* __restrict__ router, int T, int E, int K, int top,
                                                              int renorm, float wscale) {
  __shared__ __attribute__((aligned(16))) float part[RNW][EB][64][4];
  const int w = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int lr = lane & 15, lg = lane >> 4;
  const int t0 = blockIdx.x * 16;
  const uint16_t* hp = h + (size_t)min(t0 + lr, T - 1) * h_stride;
  const uint16_t* rp[EB];
#pragma unroll
  for (int b = 0; b < EB; ++b) rp[b] = router + (size_t)min(16 * b + lr, E - 1) * K;
  f32x4 acc[EB];
#pragma unroll
  for (int b = 0; b < EB; ++b) acc[b] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int steps = (K + 31) >> 5, per = (steps + RNW - 1) / RNW;
  const int s_hi = min(steps, (w + 1) * per);
  const u32x4 zero = {0u, 0u, 0u, 0u};
  constexpr int U = EB <= 2 ? 4 : 2;
  for (int s = w * per; s < s_hi; s += U) {
    u32x4 hf[U], rf[U][EB];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = (s + u) * 32 + 8 * lg;
      const bool ok = s + u < s_hi && k < K;
      hf[u] = ok ? *reinterpret_cast<const u32x4*>(hp + k) : zero;
#pragma unroll
      for (int b = 0; b < EB; ++b) rf[u][b] = ok ? *reinterpret_cast<const u32x4*>(rp[b] + k) : zero;
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int b = 0; b < EB; ++b)
        acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(rf[u][b]), as_bf16x8(hf[u]), acc[b], 0, 0, 0);
  }
#pragma unroll
  for (int b = 0; b < EB; ++b) *reinterpret_cast<f32x4*>(part[w][b][lane]) = acc[b];
  __syncthreads();
  // expert 16 b + 4 g + i of token j sits at part[.][b][16 g + j][i]; lane l of a wave takes expert l
  static_assert(RNW == 16, "one wave per token");
  const int j = w, t = t0 + j;
  if (t >= T) return;                                  // no barrier follows
  float z = -__builtin_inff();
  if (lane < E) {
    z = 0.f;
#pragma unroll
    for (int ww = 0; ww < RNW; ++ww) z += part[ww][lane >> 4][((lane >> 2) & 3) * 16 + j][lane & 3];
  }
  const float s = lane < E ? 1.f / (1.f + expf(-z)) : 0.f;
  float c = lane < E ? s : -__builtin_inff();
  float sum = 0.f, mine = 0.f;
  int slot = -1;
  for (int k = 0; k < top; ++k) {
    float bv = c;
    int bi = lane;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(bv, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (ov > bv || (ov == bv && oi < bi)) { bv = ov; bi = oi; }
    }
    if (lane == bi) { slot = k; mine = s; c = -__builtin_inff(); }
    sum += bv;
  }
  if (slot >= 0) {
    idx[(size_t)t * top + slot] = lane;
    wts[(size_t)t * top + slot] = mine * (renorm ? 1.f / (sum + 1e-20f) : 1.f) * wscale;
  }
}

}  // namespace

// h [T, K] bf16, router [E, K] bf16, E <= 64; K a multiple of 8
extern "C" int dgi_moe_router(int* idx, float* wts, const void* h, int h_stride, const void* router, int T, int E, int K, int top,
                              int renorm, float wscale, hipStream_t s) {
  if (T == 0) return 0;
  if (E < 1 || E > 64 || top < 1 || top > E || K < 8 || K % 8 || h_stride % 8 || (((uintptr_t)h | (uintptr_t)router) & 15)) return -2;
  const int grid = (T + 15) / 16;
#define DGI_RT(EB_)                                                                                                          \
  moe_router_kernel<EB_><<<grid, 64 * RNW, 0, s>>>(idx, wts, (const uint16_t*)h, h_stride, (const uint16_t*)router, T, E, K, top, \
                                                   renorm, wscale)
  if (E <= 16) DGI_RT(1);
  else if (E <= 32) DGI_RT(2);
  else if (E <= 48) DGI_RT(3);
  else DGI_RT(4);
#undef DGI_RT
  DGI_CHECK_LAUNCH();
  return 0;
}

extern "C" int dgi_moe_plan(const int* idx, int P, int E, int* order, int* where, int* seg, hipStream_t s) {
  if (E <= 0) return -2;
  moe_plan_kernel<<<E, PLAN_NT, 0, s>>>(idx, P, E, order, where, seg);
  DGI_CHECK_LAUNCH();
  return 0;
}

// glu: b [E, 2 N, K] and order / top (and pair_scale) map a place to its row of a; else b [E, N, K] and row = place.
// rows_per_tile: 16, 32, 64 (few rows per expert) or 128.  places: the most places seg can hold.
extern "C" int dgi_moe_group(const void* a, int a_stride, const void* b, void* out, const int* seg, const int* order,
                             const float* pair_scale, int places, int E, int N, int K, int top, int glu, int act, float limit,
                             float alpha, int rows_per_tile, hipStream_t s) {
  if (places == 0 || N == 0) return 0;
  if (K <= 0 || K % 8 || a_stride % 8 || (((uintptr_t)a | (uintptr_t)b) & 15) || E <= 0 || (glu && (!order || top <= 0))) return -2;
  GroupArgs g{(const uint16_t*)a, a_stride, (const uint16_t*)b, (uint16_t*)out, seg, glu ? order : nullptr, pair_scale,
              E, N, K, top, act, limit, alpha, 0};
  const int rc = glu ? launch_group<true>(g, places, rows_per_tile, s) : launch_group<false>(g, places, rows_per_tile, s);
  if (rc) return rc;
  DGI_CHECK_LAUNCH();
  return 0;
}
