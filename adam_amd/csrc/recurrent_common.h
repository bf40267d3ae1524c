// What the sequence mixers with a matrix state share: sizes, and the short convolution ahead of the recurrence.
//
// The convolution's inputs of the last `taps` tokens live in a ring of `taps` places per sequence, token p at place
// p % taps: a step reads the places of the taps - 1 tokens before its own and writes its own, so workgroups need no order.
#pragma once
#include "linear_common.h"

namespace adamah {

#define CH 16u            // tokens of a chunk
#define MAX_TAPS 16       // of the short convolution
#define VC 32u            // value columns of a decode workgroup
#define NO_MEMORY 110.0f  // exp(-110) is zero in float32: a stronger decay per token changes nothing, and the sums stay small

__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float wave_add(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}
// silu of the causal convolution at token position p for channel ch, older inputs from the ring only.  The taps' loads do
// not depend on each other: up to TM of them are asked for at once (TM >= taps).
template <int TM>
__device__ __forceinline__ float conv_silu_ring(const float* x, const float* ring, uint32_t n_ch, uint32_t ch, uint32_t p,
                                                const float* w, uint32_t taps, float bias = 0.f) {
  float in[TM], wt[TM];
#pragma unroll
  for (int j = 0; j < TM; j++) {
    const bool on = (uint32_t)j < taps && (uint32_t)j <= p;
    in[j] = !on ? 0.f : j == 0 ? x[ch] : ring[(uint64_t)((p - (uint32_t)j) % taps) * n_ch + ch];
    wt[j] = on ? w[taps - 1u - (uint32_t)j] : 0.f;
  }
  float a = bias;
#pragma unroll
  for (int j = 0; j < TM; j++) a = fmaf(wt[j], in[j], a);
  return silu_f(a);
}
// The same for CH consecutive tokens of a portion: rows r0 .. r0 + CH - 1 of x (zero results from row m on), row 0 at
// position pos; put(t, value).
template <int TM, class Put>
__device__ __forceinline__ void conv_silu_rows(const float* x, uint32_t x_stride, uint32_t r0, uint32_t m, const float* ring, uint32_t n_ch,
                                               uint32_t ch, uint32_t pos, const float* w, uint32_t taps, Put put, float bias = 0.f) {
  float in[CH + TM - 1], wt[TM];
#pragma unroll
  for (int i = 0; i < (int)CH + TM - 1; i++) {
    const int64_t r = (int64_t)r0 + i - (TM - 1);
    const bool old = r < 0, on = old ? (uint32_t)-r < taps && (uint32_t)-r <= pos : r < (int64_t)m;
    in[i] = !on ? 0.f : old ? ring[(uint64_t)((pos + (uint32_t)r) % taps) * n_ch + ch] : x[(uint64_t)r * x_stride + ch];
  }
#pragma unroll
  for (int j = 0; j < TM; j++) wt[j] = (uint32_t)j < taps ? w[taps - 1u - (uint32_t)j] : 0.f;
#pragma unroll
  for (int t = 0; t < (int)CH; t++) {
    float a = bias;
#pragma unroll
    for (int j = 0; j < TM; j++) a = fmaf(wt[j], in[t + TM - 1 - j], a);
    put(t, r0 + (uint32_t)t < m ? silu_f(a) : 0.f);
  }
}

}  // namespace adamah
