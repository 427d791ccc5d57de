// dgi/csrc/mix/embed_sinusoid.hip — token embedding of models whose positions are a sinusoidal vector:
//
//     x[t][c] = table[id_t][c] * scale + (c even ? sin : cos)(p_t * freq[c])
//
// The angle is the fp64 product of the position and the frequency, reduced to one turn in fp64, so the fp32 sine and
// cosine see a small, exact argument at any position.  One workgroup per row; x is the fp32 residual stream.
#include "../common.h"

using namespace dgi;

namespace {

template <typename T>
__global__ __launch_bounds__(256) void embed_sinusoid_kernel(float* __restrict__ x, const int* __restrict__ ids,
                                                             const int* __restrict__ positions, const T* __restrict__ table,
                                                             int vocab, float scale, const double* __restrict__ freqs, int W) {
  const int t = blockIdx.x;
  const int id = min(max(ids[t], 0), vocab - 1);
  const double p = (double)positions[t];
  for (int c = threadIdx.x; c < W; c += 256) {
    double a = p * freqs[c];
    a -= rint(a * 0.15915494309189535) * 6.283185307179586;
    float sn, cs;
    sincosf((float)a, &sn, &cs);
    float e;
    if constexpr (sizeof(T) == 2) e = bf16_to_f32(table[(size_t)id * W + c]);
    else e = table[(size_t)id * W + c];
    x[(size_t)t * W + c] = e * scale + ((c & 1) ? cs : sn);
  }
}

}  // namespace

extern "C" int dgi_embed_sinusoid(float* x, const int* ids, const int* positions, const void* table, int vocab, float scale,
                                  const double* freqs, int T, int W, int is_f32, hipStream_t s) {
  if (T == 0 || W == 0) return 0;
  if (vocab <= 0) return -2;
  if (is_f32)
    embed_sinusoid_kernel<float><<<T, 256, 0, s>>>(x, ids, positions, (const float*)table, vocab, scale, freqs, W);
  else
    embed_sinusoid_kernel<uint16_t><<<T, 256, 0, s>>>(x, ids, positions, (const uint16_t*)table, vocab, scale, freqs, W);
  DGI_CHECK_LAUNCH();
  return 0;
}
