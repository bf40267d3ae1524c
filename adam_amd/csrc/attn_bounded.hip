// Softmax attention over a bounded run of keys, without rotation, in two forms:
//   chunk    inside fixed chunks of the sequence, a logarithmic distance penalty, values divided by their root mean square
//   window   over a sliding window: unit queries and keys, a query temperature, capped scores, a linear distance penalty,
//            a sink per head in the denominator
//
// A token at position i sees positions floor(i / C) C .. i, or i - C + 1 .. i, so the cache of a sequence is C places per
// layer, token i at place i % C; what a later token overwrites is never seen again.  What is normed is cached normed.
//
// One token: k_attn_step, a workgroup per key head (or RG of its query heads) and span of places, every key and value
// read once for all of them; the token's own key and value come from the projections, and the workgroup whose span holds
// its place stores them.  More than one span: k_attn_join.
//
// A portion of a prompt: k_attn_stage lays the keys the portion sees -- what the cache holds that its first token sees,
// then the portion's own -- out as matrix operands, K [np, dp] and V transposed [vp, np]; k_attn_keep then brings the
// cache up to date; k_attn_f32 / _bf16 take 16 queries of a head per wave through the keys they see.
// Scores arrive as K . Q^T, so a lane holds four keys of one query, which is also the layout the second
// product wants its right operand in: no shared memory.  float32: the float32 matrix instruction throughout.  bfloat16:
// keys and values rounded once, queries and softmax weights as sums of two bfloat16 terms, all sums in float32.
// Scores, penalties, caps and weights are float32 in both.
#include "linear_common.h"
#include <algorithm>

namespace adamah {

// What the kernels take, from either spec.  size: chunk or window.  p1, p2: chunk: the penalty's two factors per head,
// window: slope and sink per head.
struct ASpec {
  uint32_t heads, kv_heads, dim, vdim, size, x, x_stride, x_q, x_k, x_v, p1, p2;
  float scale, eps;
  uint32_t out, out_stride, k_off, v_off, seq_stride, has_sink, qk_norm, temp_every;
  float softcap, temp_coef;
};
#define MAX_SPANS 64u
#define STEP_WAVES 8u     // of a workgroup that decodes one token
#define LOG2E 1.44269504f
#define ATT_MASKED (-1.0e30f)

// What a query of the window form is multiplied by beside its own length.
__device__ __forceinline__ float query_temperature(const ASpec& s, uint32_t p) {
  return s.temp_coef == 0.f ? 1.0f : fmaf(s.temp_coef, logf((float)((p + 1u) / s.temp_every + 1u)), 1.0f);
}
// Eight consecutive elements as they are stored, and as numbers.
template <class T> struct Eight;
template <> struct Eight<float> {
  float4 a, b;
  __device__ __forceinline__ void zero() { a = b = make_float4(0, 0, 0, 0); }
  __device__ __forceinline__ void load(const float* p) { a = *(const float4*)p; b = *(const float4*)(p + 4); }
  __device__ __forceinline__ void set(const float (&x)[8]) { a = make_float4(x[0], x[1], x[2], x[3]); b = make_float4(x[4], x[5], x[6], x[7]); }
  __device__ __forceinline__ void get(float (&o)[8]) const { o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w; o[4] = b.x; o[5] = b.y; o[6] = b.z; o[7] = b.w; }
};
template <> struct Eight<bf16_t> {
  uint4 a;
  __device__ __forceinline__ void zero() { a = make_uint4(0, 0, 0, 0); }
  __device__ __forceinline__ void load(const bf16_t* p) { a = *(const uint4*)p; }
  __device__ __forceinline__ void set(const float (&x)[8]) {
    union { bf8_t v; uint4 u; } c;
#pragma unroll
    for (int i = 0; i < 8; i++) c.v[i] = (bf16_t)x[i];
    a = c.u;
  }
  __device__ __forceinline__ void get(float (&o)[8]) const {
    o[0] = bf_lo(a.x); o[1] = bf_hi(a.x); o[2] = bf_lo(a.y); o[3] = bf_hi(a.y);
    o[4] = bf_lo(a.z); o[5] = bf_hi(a.z); o[6] = bf_lo(a.w); o[7] = bf_hi(a.w);
  }
};

// cap * tanh(a), the cap in powers of two; bfloat16: by one exponential (an error of 1e-7 of the cap)
template <class T> __device__ __forceinline__ float capped(float a, float cap) {
  if (sizeof(T) == 4) return cap * tanhf(a);
  return fmaf(-2.0f * cap, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(a * (2.0f * LOG2E)) + 1.0f), cap);
}

// ---- one token ------------------------------------------------------------------------------------------------------
// grid (key heads * groups of RG query heads, spans, sequences).  Sixteen lanes share a key: lane l16 holds columns
// 8 l16 + 128 c; a wave takes 4 KI keys at a time, their keys and values asked for together.  part: per (sequence, head,
// span) vdim + 2 floats {max in powers of two, sum, values}, used when there is more than one span.
template <class T, bool WIN, int NC, int RG, int KI>
__global__ void __launch_bounds__(STEP_WAVES * 64)
k_attn_step(const ASpec s, float* act, T* cache, float* part, uint32_t seq0, uint32_t pos, uint32_t span, uint32_t parts) {
  __shared__ float qb[RG][128 * NC];
  __shared__ float ob[STEP_WAVES][RG][128 * NC], ml[STEP_WAVES][RG][2], qi[RG];
  const uint32_t D = s.dim, V = s.vdim, D8 = (D + 7u) & ~7u, V8 = (V + 7u) & ~7u, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
  const uint32_t row = blockIdx.z, rep = s.heads / s.kv_heads, kv = blockIdx.x / parts, h0 = kv * rep + (blockIdx.x - kv * parts) * RG;
  const uint32_t nh = min((uint32_t)RG, (kv + 1u) * rep - h0);       // query heads of this workgroup
  const uint32_t me = pos % s.size, n = WIN ? min(pos + 1u, s.size) : me + 1u;       // the token's place; places in use
  const uint32_t k0 = blockIdx.y * span, k1 = min(n, k0 + span), l16 = lane & 15u, kq = lane >> 4;
  const float* x = act + s.x + (uint64_t)row * s.x_stride;
  const float* xk = x + s.x_k + kv * D;
  const float* xv = x + s.x_v + kv * V;
  T* K = cache + (uint64_t)(seq0 + row) * s.seq_stride + s.k_off + (uint64_t)kv * s.size * D8;
  T* Vc = cache + (uint64_t)(seq0 + row) * s.seq_stride + s.v_off + (uint64_t)kv * s.size * V8;
  const bool own = me >= k0 && me < k1;                         // this span holds the token's place
  Eight<T> kr[KI][NC], vr[KI][NC];
  auto fetch = [&](uint32_t kb) {
#pragma unroll
    for (int j = 0; j < KI; j++) {
      const uint32_t key = kb + kq + 4u * j;
#pragma unroll
      for (int c = 0; c < NC; c++) {
        const uint32_t d = l16 * 8u + 128u * c;
        kr[j][c].zero(); vr[j][c].zero();
        if (key != me && key < k1) {
          if (d < D8) kr[j][c].load(K + (uint64_t)key * D8 + d);
          if (d < V8) vr[j][c].load(Vc + (uint64_t)key * V8 + d);
        }
      }
    }
  };
  fetch(k0 + wave * 4u * KI);                                   // the first keys are on their way while the queries are staged
  float iv = 1.f, ik = 1.f;
  if (own && !WIN) {
    iv = 0.f;
    for (uint32_t d = lane; d < V; d += 64u) iv = fmaf(xv[d], xv[d], iv);
    iv = 1.0f / sqrtf(wsum64(iv) / (float)V + s.eps);
  }
  if (own && WIN && s.qk_norm) {
    ik = 0.f;
    for (uint32_t d = lane; d < D; d += 64u) ik = fmaf(xk[d], xk[d], ik);
    ik = 1.0f / sqrtf(wsum64(ik) / (float)D + s.eps);
  }
  if (WIN && wave < nh) {                                       // a wave per query head: what its scores are multiplied by
    const float* xq = x + s.x_q + (h0 + wave) * D;
    float f = s.scale * query_temperature(s, pos);
    if (s.qk_norm) {
      float a = 0.f;
      for (uint32_t d = lane; d < D; d += 64u) a = fmaf(xq[d], xq[d], a);
      f /= sqrtf(wsum64(a) / (float)D + s.eps);
    }
    if (lane == 0) qi[wave] = s.softcap > 0.f ? f / s.softcap : f * LOG2E;
  }
  for (uint32_t i = tid; i < RG * 128u * NC; i += STEP_WAVES * 64u) {
    const uint32_t r = i / (128u * NC), d = i - r * (128u * NC);
    qb[r][d] = (r < nh && d < D) ? x[s.x_q + (h0 + r) * D + d] * (WIN ? 1.0f : s.scale * LOG2E) : 0.f;
  }
  float r1[RG], r2[RG], mx[RG], sum[RG], o[RG][NC][8];
#pragma unroll
  for (int r = 0; r < RG; r++) {
    const uint32_t h = h0 + min((uint32_t)r, nh - 1u);
    r1[r] = act[s.p1 + h] * (WIN ? LOG2E : 1.0f); r2[r] = WIN ? 0.f : act[s.p2 + h];
    mx[r] = ATT_MASKED; sum[r] = 0.f;
#pragma unroll
    for (int c = 0; c < NC; c++)
#pragma unroll
      for (int i = 0; i < 8; i++) o[r][c][i] = 0.f;
  }
  __syncthreads();
  for (uint32_t kb = k0 + wave * 4u * KI; kb < k1; kb += STEP_WAVES * 4u * KI) {
    if (kb >= k0 + STEP_WAVES * 4u * KI) fetch(kb);
    if (own && me - kb < 4u * KI) {                         // the token's own key and value
#pragma unroll
      for (int j = 0; j < KI; j++)
        if (kb + kq + 4u * j == me) {
#pragma unroll
          for (int c = 0; c < NC; c++) {
            const uint32_t d = l16 * 8u + 128u * c;
            float a[8], b[8];
#pragma unroll
            for (int i = 0; i < 8; i++) { a[i] = d + i < D ? xk[d + i] * ik : 0.f; b[i] = d + i < V ? xv[d + i] * iv : 0.f; }
            kr[j][c].set(a); vr[j][c].set(b);
          }
        }
    }
    float kk[KI][NC][8], vv[KI][NC][8];
#pragma unroll
    for (int j = 0; j < KI; j++)
#pragma unroll
      for (int c = 0; c < NC; c++) { kr[j][c].get(kk[j][c]); vr[j][c].get(vv[j][c]); }
#pragma unroll
    for (int r = 0; r < RG; r++) {
      float sc[KI], top = ATT_MASKED;
#pragma unroll
      for (int j = 0; j < KI; j++) sc[j] = 0.f;
#pragma unroll
      for (int c = 0; c < NC; c++) {
        float q[8];
#pragma unroll
        for (int i = 0; i < 8; i++) q[i] = qb[r][128u * c + l16 * 8u + i];
#pragma unroll
        for (int j = 0; j < KI; j++)
#pragma unroll
          for (int i = 0; i < 8; i++) sc[j] = fmaf(kk[j][c][i], q[i], sc[j]);
      }
#pragma unroll
      for (int j = 0; j < KI; j++) {
        float a = row16_sum(sc[j]);
        const uint32_t key = kb + kq + 4u * j;
        if (WIN) {
          a *= qi[r];
          if (s.softcap > 0.f) a = capped<T>(a, s.softcap * LOG2E);
          sc[j] = key < k1 ? a - r1[r] * (float)(key <= me ? me - key : me + s.size - key) : ATT_MASKED;
        } else
          sc[j] = key < k1 ? a - r1[r] * __builtin_amdgcn_logf(fmaf(r2[r], (float)(me - key), 1.0f)) : ATT_MASKED;
        top = fmaxf(top, sc[j]);
      }
      top = fmaxf(top, __shfl_xor(top, 16, 64)); top = fmaxf(top, __shfl_xor(top, 32, 64));
      const float nm = fmaxf(mx[r], top), al = __builtin_amdgcn_exp2f(mx[r] - nm);
      mx[r] = nm;
      sum[r] *= al;
#pragma unroll
      for (int c = 0; c < NC; c++)
#pragma unroll
        for (int i = 0; i < 8; i++) o[r][c][i] *= al;
#pragma unroll
      for (int j = 0; j < KI; j++) {
        const float p = sc[j] > 0.5f * ATT_MASKED ? __builtin_amdgcn_exp2f(sc[j] - nm) : 0.f;
        sum[r] += p;
#pragma unroll
        for (int c = 0; c < NC; c++)
#pragma unroll
          for (int i = 0; i < 8; i++) o[r][c][i] = fmaf(p, vv[j][c][i], o[r][c][i]);
      }
    }
  }
#pragma unroll
  for (int r = 0; r < RG; r++) {                                // the four key groups of a wave, then the waves
    sum[r] += __shfl_xor(sum[r], 16, 64); sum[r] += __shfl_xor(sum[r], 32, 64);
    if (lane == 0) { ml[wave][r][0] = mx[r]; ml[wave][r][1] = sum[r]; }
#pragma unroll
    for (int c = 0; c < NC; c++)
#pragma unroll
      for (int i = 0; i < 8; i++) {
        float a = o[r][c][i];
        a += __shfl_xor(a, 16, 64); a += __shfl_xor(a, 32, 64);
        if (kq == 0) ob[wave][r][128u * c + l16 * 8u + i] = a;
      }
  }
  __syncthreads();
  for (uint32_t i = tid; i < nh * V; i += STEP_WAVES * 64u) {
    const uint32_t r = i / V, d = i - r * V, h = h0 + r;
    float m4 = ml[0][r][0];
#pragma unroll
    for (uint32_t w = 1; w < STEP_WAVES; w++) m4 = fmaxf(m4, ml[w][r][0]);
    float a = 0.f, t = 0.f;
#pragma unroll
    for (uint32_t w = 0; w < STEP_WAVES; w++) { const float e = __builtin_amdgcn_exp2f(ml[w][r][0] - m4); a = fmaf(e, ob[w][r][d], a); t = fmaf(e, ml[w][r][1], t); }
    if (WIN && s.has_sink && gridDim.y == 1) {
      const float sk = act[s.p2 + h] * LOG2E, top = fmaxf(m4, sk), e = __builtin_amdgcn_exp2f(m4 - top);
      a *= e; t = fmaf(t, e, __builtin_amdgcn_exp2f(sk - top));
    }
    if (gridDim.y == 1) act[s.out + (uint64_t)row * s.out_stride + h * V + d] = a / t;
    else {
      float* p = part + (((uint64_t)row * s.heads + h) * gridDim.y + blockIdx.y) * (V + 2u);
      p[2u + d] = a;
      if (d == 0) { p[0] = m4; p[1] = t; }
    }
  }
  if (own && h0 == kv * rep) {
    for (uint32_t d = tid; d < D8; d += STEP_WAVES * 64u) K[(uint64_t)me * D8 + d] = (T)(d < D ? xk[d] * ik : 0.f);
    for (uint32_t d = tid; d < V8; d += STEP_WAVES * 64u) Vc[(uint64_t)me * V8 + d] = (T)(d < V ? xv[d] * iv : 0.f);
  }
}
__global__ void __launch_bounds__(256)
k_attn_join(const ASpec s, float* act, const float* __restrict__ part, uint32_t n_part) {
  __shared__ float w[MAX_SPANS];
  const uint32_t h = blockIdx.x, row = blockIdx.y, V = s.vdim, lane = threadIdx.x;
  const float* p = part + ((uint64_t)row * s.heads + h) * n_part * (V + 2u);
  if (lane < 64u) {
    const float m = lane < n_part ? p[(uint64_t)lane * (V + 2u)] : ATT_MASKED, l = lane < n_part ? p[(uint64_t)lane * (V + 2u) + 1u] : 0.f;
    const float sk = s.has_sink ? act[s.p2 + h] * LOG2E : ATT_MASKED;
    float mx = fmaxf(m, sk);
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
    const float e = lane < n_part ? __builtin_amdgcn_exp2f(m - mx) : 0.f;
    w[lane] = e / (wsum64(e * l) + (s.has_sink ? __builtin_amdgcn_exp2f(sk - mx) : 0.f));
  }
  __syncthreads();
  for (uint32_t d = threadIdx.x; d < V; d += 256u) {
    float a = 0.f;
#pragma unroll 8
    for (uint32_t i = 0; i < n_part; i++) a = fmaf(w[i], p[(uint64_t)i * (V + 2u) + 2u + d], a);
    act[s.out + (uint64_t)row * s.out_stride + h * V + d] = a;
  }
}

// ---- a portion ------------------------------------------------------------------------------------------------------
struct StageDims { uint32_t past, n, np, dp, vp, place0; };   // keys from the cache, keys in all, padded counts, first key's place
// One workgroup per 32 staged keys and key head.  K: [kv_heads, np, dp], VT: [kv_heads, vp, np].
template <class T, bool WIN>
__global__ void __launch_bounds__(256)
k_attn_stage(const ASpec s, const float* __restrict__ act, const T* cache, T* __restrict__ K, T* __restrict__ VT, StageDims sd) {
  extern __shared__ float vt[];                    // [32][V + 1]
  __shared__ float inv[32];
  const uint32_t D = s.dim, V = s.vdim, D8 = (D + 7u) & ~7u, V8 = (V + 7u) & ~7u, tid = threadIdx.x, kv = blockIdx.y, j0 = blockIdx.x * 32u;
  const T* cK = cache + s.k_off + (uint64_t)kv * s.size * D8;
  const T* cV = cache + s.v_off + (uint64_t)kv * s.size * V8;
  const float* xk = act + s.x + s.x_k + kv * D;
  const float* xv = act + s.x + s.x_v + kv * V;
  {                                                // root mean squares of the new values (window: keys): 8 threads a key
    const uint32_t j = j0 + (tid >> 3), len = WIN ? D : V;
    float ss = 0.f;
    if (j >= sd.past && j < sd.n)
      for (uint32_t d = tid & 7u; d < len; d += 8u) { const float v = (WIN ? xk : xv)[(uint64_t)(j - sd.past) * s.x_stride + d]; ss = fmaf(v, v, ss); }
    ss += __shfl_xor(ss, 1, 64); ss += __shfl_xor(ss, 2, 64); ss += __shfl_xor(ss, 4, 64);
    if ((tid & 7u) == 0) inv[tid >> 3] = !WIN || s.qk_norm ? 1.0f / sqrtf(ss / (float)len + s.eps) : 1.0f;
  }
  __syncthreads();
  for (uint32_t i = tid; i < 32u * sd.dp; i += 256u) {
    const uint32_t jj = i / sd.dp, d = i - jj * sd.dp, j = j0 + jj;
    T v = (T)0.f;
    if (d < D && j < sd.n) v = j < sd.past ? cK[(uint64_t)((sd.place0 + j) % s.size) * D8 + d] : (T)(xk[(uint64_t)(j - sd.past) * s.x_stride + d] * (WIN ? inv[jj] : 1.0f));
    K[((uint64_t)kv * sd.np + j) * sd.dp + d] = v;
  }
  for (uint32_t i = tid; i < 32u * V; i += 256u) {
    const uint32_t jj = i / V, d = i - jj * V, j = j0 + jj;
    float v = 0.f;
    if (j < sd.n) v = j < sd.past ? (float)cV[(uint64_t)((sd.place0 + j) % s.size) * V8 + d] : xv[(uint64_t)(j - sd.past) * s.x_stride + d] * (WIN ? 1.0f : inv[jj]);
    vt[jj * (V + 1u) + d] = v;
  }
  __syncthreads();
  for (uint32_t i = tid; i < 32u * sd.vp; i += 256u) {
    const uint32_t d = i >> 5, jj = i & 31u;
    VT[((uint64_t)kv * sd.vp + d) * sd.np + j0 + jj] = (T)(d < V ? vt[jj * (V + 1u) + d] : 0.f);
  }
}
// The cache after the portion: the tokens a later one may see.  A launch of its own, behind the staging that
// still reads the places it writes.
template <class T>
__global__ void __launch_bounds__(256)
k_attn_keep(const ASpec s, T* cache, const T* __restrict__ K, const T* __restrict__ VT, StageDims sd, uint32_t first) {
  const uint32_t D8 = (s.dim + 7u) & ~7u, V8 = (s.vdim + 7u) & ~7u, kv = blockIdx.y, j = first + blockIdx.x;
  const uint32_t place = (sd.place0 + j) % s.size;
  T* cK = cache + s.k_off + ((uint64_t)kv * s.size + place) * D8;
  T* cV = cache + s.v_off + ((uint64_t)kv * s.size + place) * V8;
  for (uint32_t d = threadIdx.x; d < D8; d += 256u) cK[d] = K[((uint64_t)kv * sd.np + j) * sd.dp + d];
  for (uint32_t d = threadIdx.x; d < V8; d += 256u) cV[d] = VT[((uint64_t)kv * sd.vp + d) * sd.np + j];
}

// First staged key that the query at position p sees; base: position of the first staged key.
template <bool WIN> __device__ __forceinline__ uint32_t first_seen(const ASpec& s, uint32_t p, uint32_t base) {
  return (WIN ? (p >= s.size ? p + 1u - s.size : 0u) : p / s.size * s.size) - base;
}
// 16 queries of a head per wave.  float32 form: keys 16 at a time.
template <bool WIN, int NV>
__global__ void __launch_bounds__(256)
k_attn_f32(const ASpec s, float* act, const float* __restrict__ K, const float* __restrict__ VT, StageDims sd, uint32_t m, uint32_t pos) {
  const uint32_t lane = threadIdx.x & 63u, c = lane & 15u, kg = lane >> 4, h = blockIdx.x, kv = h / (s.heads / s.kv_heads);
  const uint32_t q0 = (blockIdx.y * 4u + (threadIdx.x >> 6)) * 16u;
  if (q0 >= m) return;
  const uint32_t qr = min(q0 + c, m - 1u), base = pos - sd.past;           // key j of the stage sits at position base + j
  const uint32_t qj = sd.past + qr, lo = first_seen<WIN>(s, pos + qr, base);   // visible: lo .. qj
  const uint32_t first = first_seen<WIN>(s, pos + q0, base) & ~15u, end = sd.past + min(q0 + 16u, m);
  const float* xq = act + s.x + (uint64_t)qr * s.x_stride + s.x_q + h * s.dim;
  const float* kb = K + (uint64_t)kv * sd.np * sd.dp;
  const float* vb = VT + (uint64_t)kv * sd.vp * sd.np;
  const float r1 = act[s.p1 + h], r2 = act[s.p2 + h];
  f4_t o[NV];
#pragma unroll
  for (int i = 0; i < NV; i++) o[i] = (f4_t){0, 0, 0, 0};
  float mx = ATT_MASKED, sum = 0.f, qs = s.scale;
  if (WIN) {
    if (s.has_sink) { mx = r2; sum = 1.f; }
    if (s.qk_norm) {
      float a = 0.f;
      for (uint32_t d = kg; d < s.dim; d += 4u) a = fmaf(xq[d], xq[d], a);
      a += __shfl_xor(a, 16, 64); a += __shfl_xor(a, 32, 64);
      qs /= sqrtf(a / (float)s.dim + s.eps);
    }
    qs *= query_temperature(s, pos + qr);
  }
  for (uint32_t j0 = first; j0 < end; j0 += 16u) {
    f4_t a = {0, 0, 0, 0};
    for (uint32_t d0 = 0; d0 < sd.dp; d0 += 16u) {
      const f4_t kk = *(const f4_t*)(kb + (uint64_t)(j0 + c) * sd.dp + d0 + 4u * kg);
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const uint32_t d = d0 + 4u * kg + i;
        a = __builtin_amdgcn_mfma_f32_16x16x4f32(kk[i], d < s.dim ? xq[d] : 0.f, a, 0, 0, 0);
      }
    }
    float t = ATT_MASKED;
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const uint32_t j = j0 + 4u * kg + i;
      const bool ok = j >= lo && j <= qj;
      if (WIN) {
        float z = a[i] * qs;
        if (s.softcap > 0.f) z = s.softcap * tanhf(z / s.softcap);
        a[i] = ok ? z - r1 * (float)(qj - j) : ATT_MASKED;
      } else
        a[i] = ok ? a[i] * s.scale - r1 * log1pf(r2 * (float)(qj - j)) : ATT_MASKED;
      t = fmaxf(t, a[i]);
    }
    t = fmaxf(t, __shfl_xor(t, 16, 64)); t = fmaxf(t, __shfl_xor(t, 32, 64));
    const float nm = fmaxf(mx, t), al = expf(mx - nm);
    mx = nm;
    float ps = 0.f;
#pragma unroll
    for (int i = 0; i < 4; i++) { a[i] = a[i] > 0.5f * ATT_MASKED ? expf(a[i] - nm) : 0.f; ps += a[i]; }
    ps += __shfl_xor(ps, 16, 64); ps += __shfl_xor(ps, 32, 64);
    sum = fmaf(sum, al, ps);
#pragma unroll
    for (int v = 0; v < NV; v++) {
      if ((uint32_t)v * 16u >= sd.vp) break;
      const f4_t vv = *(const f4_t*)(vb + (uint64_t)(v * 16u + c) * sd.np + j0 + 4u * kg);
      o[v] *= al;
#pragma unroll
      for (int i = 0; i < 4; i++) o[v] = __builtin_amdgcn_mfma_f32_16x16x4f32(vv[i], a[i], o[v], 0, 0, 0);
    }
  }
  if (q0 + c >= m) return;
  float* out = act + s.out + (uint64_t)qr * s.out_stride + h * s.vdim;
#pragma unroll
  for (int v = 0; v < NV; v++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const uint32_t d = v * 16u + 4u * kg + i;
      if (d < s.vdim) out[d] = o[v][i] / sum;
    }
}

// bfloat16 form: QT tiles of 16 queries a wave, keys 32 at a time (two tiles of 16); DK: k-steps of 32 dimensions.  Scores
// and the penalty are kept in powers of two.  A step's values and the next step's keys are in flight under the products.
template <bool WIN, int DK, int NV, int QT>
__global__ void __launch_bounds__(256, DK * QT <= 8 && NV * QT <= 16 ? 2 : 1)
k_attn_bf16(const ASpec s, float* act, const bf16_t* __restrict__ K, const bf16_t* __restrict__ VT, StageDims sd, uint32_t m, uint32_t pos) {
  // workgroups land on the eight dies in turn: the query heads of a key head share one; late query tiles, which see more
  // keys, go with early ones
  const uint32_t nx = gridDim.x, h = (nx & 7u) == 0u ? (blockIdx.x & 7u) * (nx >> 3) + (blockIdx.x >> 3) : blockIdx.x;
  const uint32_t ny = gridDim.y, by = blockIdx.y < (ny >> 1) ? blockIdx.y : ny - 1u - (blockIdx.y - (ny >> 1));
  const uint32_t lane = threadIdx.x & 63u, c = lane & 15u, kg = lane >> 4, kv = h / (s.heads / s.kv_heads);
  const uint32_t q0 = (by * 4u + (threadIdx.x >> 6)) * 16u * QT;
  if (q0 >= m) return;
  const uint32_t base = pos - sd.past, qlast = min(q0 + 16u * QT, m) - 1u;
  const uint32_t first = first_seen<WIN>(s, pos + q0, base) & ~31u, end = sd.past + qlast + 1u;
  const uint32_t lo_all = first_seen<WIN>(s, pos + qlast, base);           // seen by every query from here to past + q0
  const bf16_t* kb = K + (uint64_t)kv * sd.np * sd.dp + (uint64_t)c * sd.dp + 8u * kg;
  const bf16_t* vb = VT + (uint64_t)kv * sd.vp * sd.np + (uint64_t)c * sd.np + 4u * kg;
  const float r1 = act[s.p1 + h] * (WIN ? LOG2E : 1.0f), r2 = act[s.p2 + h] * (WIN ? LOG2E : 1.0f);
  const float cap = WIN ? s.softcap * LOG2E : 0.f;
  uint32_t qr[QT], qj[QT], lo[QT];
  bf8_t qh[QT][DK], ql[QT][DK];
#pragma unroll
  for (int g = 0; g < QT; g++) {
    qr[g] = min(q0 + 16u * g + c, m - 1u);
    qj[g] = sd.past + qr[g];
    lo[g] = first_seen<WIN>(s, pos + qr[g], base);
    const float* xq = act + s.x + (uint64_t)qr[g] * s.x_stride + s.x_q + h * s.dim;
    float qs = s.scale * LOG2E;
    if (WIN) {                                               // capped: the exponent of the cap's own exponential
      if (s.softcap > 0.f) qs *= 2.0f / s.softcap;
      if (s.qk_norm) {
        float a = 0.f;
        for (uint32_t d = kg; d < s.dim; d += 4u) a = fmaf(xq[d], xq[d], a);
        a += __shfl_xor(a, 16, 64); a += __shfl_xor(a, 32, 64);
        qs /= sqrtf(a / (float)s.dim + s.eps);
      }
      qs *= query_temperature(s, pos + qr[g]);
    }
#pragma unroll
    for (int t = 0; t < DK; t++)
#pragma unroll
      for (int i = 0; i < 8; i++) {
        const uint32_t d = 32u * t + 8u * kg + i;
        const float x = d < s.dim ? xq[d] * qs : 0.f;
        qh[g][t][i] = (bf16_t)x;
        ql[g][t][i] = (bf16_t)(x - (float)qh[g][t][i]);
      }
  }
  f4_t o[QT][NV];
  float mx[QT], sum[QT];
#pragma unroll
  for (int g = 0; g < QT; g++) {
    mx[g] = WIN && s.has_sink ? r2 : ATT_MASKED; sum[g] = WIN && s.has_sink && kg == 0u ? 1.f : 0.f;
#pragma unroll
    for (int i = 0; i < NV; i++) o[g][i] = (f4_t){0, 0, 0, 0};
  }
  bf8_t kf[2][DK];
  auto keys = [&](uint32_t j0) {
#pragma unroll
    for (int u = 0; u < 2; u++)
#pragma unroll
      for (int t = 0; t < DK; t++) kf[u][t] = *(const bf8_t*)(kb + (uint64_t)(j0 + 16u * u) * sd.dp + 32u * t);
  };
  keys(first);
  for (uint32_t j0 = first; j0 < end; j0 += 32u) {
    bf4_t vf[NV][2];
#pragma unroll
    for (int v = 0; v < NV; v++) {
      vf[v][0] = *(const bf4_t*)(vb + (uint64_t)v * 16u * sd.np + j0);
      vf[v][1] = *(const bf4_t*)(vb + (uint64_t)v * 16u * sd.np + j0 + 16u);
    }
    f4_t a[QT][2];
#pragma unroll
    for (int g = 0; g < QT; g++)
#pragma unroll
      for (int u = 0; u < 2; u++) {
        a[g][u] = (f4_t){0, 0, 0, 0};
#pragma unroll
        for (int t = 0; t < DK; t++) {
          a[g][u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[u][t], ql[g][t], a[g][u], 0, 0, 0);
          a[g][u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[u][t], qh[g][t], a[g][u], 0, 0, 0);
        }
      }
    if (j0 + 32u < end) keys(j0 + 32u);
    const bool all = j0 >= lo_all && j0 + 31u <= sd.past + q0;
#pragma unroll
    for (int g = 0; g < QT; g++) {
      const float dist = (float)(int32_t)(qj[g] - j0 - 4u * kg);
      float t = ATT_MASKED;
#pragma unroll
      for (int u = 0; u < 2; u++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
          const float away = dist - (float)(16 * u + i), pen = r1 * (WIN ? away : __builtin_amdgcn_logf(fmaf(r2, away, 1.0f)));
          if (WIN && cap > 0.f) a[g][u][i] = fmaf(-2.0f * cap, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(a[g][u][i]) + 1.0f), cap);
          const uint32_t j = j0 + 16u * u + 4u * kg + i;
          a[g][u][i] = all || (j >= lo[g] && j <= qj[g]) ? a[g][u][i] - pen : ATT_MASKED;
          t = fmaxf(t, a[g][u][i]);
        }
      t = fmaxf(t, __shfl_xor(t, 16, 64)); t = fmaxf(t, __shfl_xor(t, 32, 64));
      const float nm = fmaxf(mx[g], t), al = __builtin_amdgcn_exp2f(mx[g] - nm);
      mx[g] = nm;
      float ps = 0.f;
      bf8_t ph, pl;
#pragma unroll
      for (int u = 0; u < 2; u++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
          const float p = all || a[g][u][i] > 0.5f * ATT_MASKED ? __builtin_amdgcn_exp2f(a[g][u][i] - nm) : 0.f;
          ps += p;
          ph[4 * u + i] = (bf16_t)p;
          pl[4 * u + i] = (bf16_t)(p - (float)ph[4 * u + i]);
        }
      sum[g] = fmaf(sum[g], al, ps);                       // per lane: the four key groups are added up at the end
#pragma unroll
      for (int v = 0; v < NV; v++) {
        const bf8_t vv = {vf[v][0][0], vf[v][0][1], vf[v][0][2], vf[v][0][3], vf[v][1][0], vf[v][1][1], vf[v][1][2], vf[v][1][3]};
        o[g][v] *= al;
        o[g][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vv, pl, o[g][v], 0, 0, 0);
        o[g][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vv, ph, o[g][v], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int g = 0; g < QT; g++) {
    sum[g] += __shfl_xor(sum[g], 16, 64); sum[g] += __shfl_xor(sum[g], 32, 64);
    if (q0 + 16u * g + c >= m) continue;
    const float inv = 1.0f / sum[g];
    float* out = act + s.out + (uint64_t)qr[g] * s.out_stride + h * s.vdim;
#pragma unroll
    for (int v = 0; v < NV; v++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const uint32_t d = v * 16u + 4u * kg + i;
        if (d < s.vdim) out[d] = o[g][v][i] * inv;
      }
  }
}

static Scratch g_stage, g_parts;
void attn_bounded_release() { scratch_free(g_stage); scratch_free(g_parts); }

template <bool WIN, int DK>
static void launch_bf16(const ASpec& s, float* act, const bf16_t* K, const bf16_t* VT, const StageDims& sd, uint32_t m, uint32_t pos) {
  switch (sd.vp / 16u) {
#define CASE(N)                                                                                                     \
  case N: {                                                                                                         \
    constexpr int QT = DK <= 4 && N <= 8 ? 2 : 1;                                                                   \
    k_attn_bf16<WIN, DK, N, QT><<<dim3(s.heads, cdiv(m, 64 * QT)), 256, 0, g.stream>>>(s, act, K, VT, sd, m, pos); \
  } break
    CASE(2); CASE(4); CASE(6); CASE(8); CASE(12); CASE(16);
#undef CASE
  }
}
static uint32_t vtiles(uint32_t v) {
  for (uint32_t t : {2u, 4u, 6u, 8u, 12u, 16u}) if (v <= 16u * t) return t;
  return 0;
}

template <class T, bool WIN>
static int run_portion(const ASpec& s, float* act, T* cache, uint32_t m, uint32_t pos) {
  StageDims sd;
  sd.past = WIN ? std::min(pos, s.size - 1u) : pos % s.size;
  sd.place0 = (pos - sd.past) % s.size;
  sd.n = sd.past + m;
  sd.np = (sd.n + 31u) & ~31u;
  sd.dp = 32u * (s.dim <= 128u ? cdiv(s.dim, 32) : s.dim <= 192u ? 6u : 8u);
  sd.vp = vtiles(s.vdim) * 16u;
  const uint64_t nk = (uint64_t)s.kv_heads * sd.np * sd.dp, nv = (uint64_t)s.kv_heads * sd.np * sd.vp;
  if (int r = scratch_need(g_stage, (nk + nv) * sizeof(T) + 64)) return r;
  T *K = (T*)g_stage.p, *VT = K + nk;
  k_attn_stage<T, WIN><<<dim3(sd.np / 32u, s.kv_heads), 256, (size_t)32 * (s.vdim + 1) * 4, g.stream>>>(s, act, cache, K, VT, sd);
  count_launch();
  if (int r = check_launch()) return r;
  // positions still wanted after the portion: the last token's chunk, or a window up to it; from its first new token on
  const uint32_t end = pos + m, from = std::max(pos, WIN ? end - std::min(end, s.size) : (end - 1u) / s.size * s.size);
  k_attn_keep<T><<<dim3(end - from, s.kv_heads), 256, 0, g.stream>>>(s, cache, K, VT, sd, from - (pos - sd.past));
  count_launch();
  if (int r = check_launch()) return r;
  if constexpr (sizeof(T) == 4) {
    const dim3 grid(s.heads, cdiv(m, 64));
    if (sd.vp <= 64u) k_attn_f32<WIN, 4><<<grid, 256, 0, g.stream>>>(s, act, K, VT, sd, m, pos);
    else k_attn_f32<WIN, 16><<<grid, 256, 0, g.stream>>>(s, act, K, VT, sd, m, pos);
  } else {
    switch (sd.dp / 32u) {
      case 1: launch_bf16<WIN, 1>(s, act, K, VT, sd, m, pos); break;
      case 2: launch_bf16<WIN, 2>(s, act, K, VT, sd, m, pos); break;
      case 3: launch_bf16<WIN, 3>(s, act, K, VT, sd, m, pos); break;
      case 4: launch_bf16<WIN, 4>(s, act, K, VT, sd, m, pos); break;
      case 6: launch_bf16<WIN, 6>(s, act, K, VT, sd, m, pos); break;
      default: launch_bf16<WIN, 8>(s, act, K, VT, sd, m, pos); break;
    }
  }
  count_launch();
  return check_launch();
}

template <class T, bool WIN, int NC, int RG, int KI>
static int run_step_as(const ASpec& s, float* act, T* cache, uint32_t n_seq, uint32_t seq0, uint32_t pos) {
  const uint32_t parts = cdiv(s.heads / s.kv_heads, RG), n = WIN ? std::min(pos + 1u, s.size) : pos % s.size + 1u, unit = STEP_WAVES * 4u * KI;
  // no more workgroups than compute units: a few too many would take as long as twice as many
  const uint32_t most = std::min<uint32_t>(MAX_SPANS, std::max<uint32_t>(1u, (uint32_t)g.n_cu / (s.kv_heads * parts * n_seq)));
  const uint32_t span = std::max<uint32_t>(unit, cdiv(cdiv(n, most), 4u * KI) * 4u * KI), spans = cdiv(n, span);
  if (s.size > unit)      // at its full size from the first step on: a graph may be recording when the second span begins
    if (int r = scratch_need(g_parts, (size_t)n_seq * s.heads * MAX_SPANS * (s.vdim + 2) * 4)) return r;
  k_attn_step<T, WIN, NC, RG, KI><<<dim3(s.kv_heads * parts, spans, n_seq), STEP_WAVES * 64, 0, g.stream>>>(s, act, cache, (float*)g_parts.p, seq0, pos, span, parts);
  count_launch();
  if (spans > 1) {
    if (int r = check_launch()) return r;
    k_attn_join<<<dim3(s.heads, n_seq), 256, 0, g.stream>>>(s, act, (const float*)g_parts.p, spans);
    count_launch();
  }
  return check_launch();
}
template <class T, bool WIN>
static int run_step(const ASpec& s, float* act, T* cache, uint32_t n_seq, uint32_t seq0, uint32_t pos) {
  const uint32_t rep = s.heads / s.kv_heads;
  constexpr int KI = 4;
#define STEP(NC, RG, K) run_step_as<T, WIN, NC, RG, K>(s, act, cache, n_seq, seq0, pos)
  if (s.dim <= 128u && s.vdim <= 128u) return rep == 1 ? STEP(1, 1, KI) : rep == 2 ? STEP(1, 2, KI) : STEP(1, 4, KI);
  return rep == 1 ? STEP(2, 1, KI / 2) : STEP(2, 2, KI / 2);
#undef STEP
}

// Ranges and sizes, then one token of each of n_seq sequences or a portion of one.
template <bool WIN>
static int run_attention(Map* ma, const ASpec& s, uint32_t cache_map, uint32_t n_seq, uint32_t rows, uint32_t seq0, uint32_t pos) {
  Map* mc = get_map(cache_map);
  if (!mc || (mc->dtype != DTYPE_F32 && mc->dtype != DTYPE_BF16)) return ADAMAH_ERR_INVALID;
  const uint64_t D = s.dim, V = s.vdim, H = s.heads, G = s.kv_heads, C = s.size, n_tok = (uint64_t)n_seq * rows;
  const uint64_t D8 = (D + 7) / 8 * 8, V8 = (V + 7) / 8 * 8;
  if (D == 0 || D > 256 || V == 0 || V > 256 || H == 0 || G == 0 || H % G || C == 0 || (uint64_t)pos + rows + C > 0xFFFFFF00ull) return ADAMAH_ERR_INVALID;
  if (s.x_q + H * D > s.x_stride || s.x_k + G * D > s.x_stride || s.x_v + G * V > s.x_stride ||
      !in_range(s.x, (n_tok - 1) * s.x_stride + s.x_stride, ma->n_elems) ||
      !in_range(s.out, (n_tok - 1) * s.out_stride + H * V, ma->n_elems) ||
      !in_range(s.p1, H, ma->n_elems) || !in_range(s.p2, H, ma->n_elems)) return ADAMAH_ERR_INVALID;
  if (((s.k_off | s.v_off | s.seq_stride) & 7u) || s.k_off + G * C * D8 > s.seq_stride || s.v_off + G * C * V8 > s.seq_stride ||
      !in_range((uint64_t)seq0 * s.seq_stride, (uint64_t)n_seq * s.seq_stride, mc->n_elems)) return ADAMAH_ERR_INVALID;
  float* act = (float*)ma->buf;
  const uint64_t slot = (uint64_t)seq0 * s.seq_stride;
  if (rows == 1)
    return mc->dtype == DTYPE_F32 ? run_step<float, WIN>(s, act, (float*)mc->buf, n_seq, seq0, pos)
                                  : run_step<bf16_t, WIN>(s, act, (bf16_t*)mc->buf, n_seq, seq0, pos);
  return mc->dtype == DTYPE_F32 ? run_portion<float, WIN>(s, act, (float*)mc->buf + slot, rows, pos)
                                : run_portion<bf16_t, WIN>(s, act, (bf16_t*)mc->buf + slot, rows, pos);
}

}  // namespace adamah

using namespace adamah;

extern "C" {

int adamah_chunk_attention_dev(uint32_t map_act, uint32_t h_spec, uint32_t n_seq, uint32_t rows, uint32_t seq0, uint32_t pos) { ADAMAH_API();
  Map* ma = get_f32_map(map_act);
  const AdamahChunkAttnSpec* s = spec_of<AdamahChunkAttnSpec>(h_spec);
  if (!ma || !s || n_seq == 0 || rows == 0 || (n_seq > 1 && rows > 1)) return ADAMAH_ERR_INVALID;
  const ASpec a = {s->heads, s->kv_heads, s->dim, s->vdim, s->chunk, s->x, s->x_stride, s->x_q, s->x_k, s->x_v, s->r1, s->r2, s->scale,
                   s->eps, s->out, s->out_stride, s->k_off, s->v_off, s->seq_stride, 0, 0, 1, 0.f, 0.f};
  return run_attention<false>(ma, a, s->cache_map, n_seq, rows, seq0, pos);
}

int adamah_window_attention_dev(uint32_t map_act, uint32_t h_spec, uint32_t n_seq, uint32_t rows, uint32_t seq0, uint32_t pos) { ADAMAH_API();
  Map* ma = get_f32_map(map_act);
  const AdamahWindowAttnSpec* s = spec_of<AdamahWindowAttnSpec>(h_spec);
  if (!ma || !s || n_seq == 0 || rows == 0 || (n_seq > 1 && rows > 1)) return ADAMAH_ERR_INVALID;
  if (s->temp_every == 0 || s->softcap < 0.f) return ADAMAH_ERR_INVALID;
  const ASpec a = {s->heads, s->kv_heads, s->dim, s->vdim, s->window, s->x, s->x_stride, s->x_q, s->x_k, s->x_v, s->slope,
                   s->has_sink ? s->sink : s->slope, s->scale, s->eps, s->out, s->out_stride, s->k_off, s->v_off, s->seq_stride,
                   s->has_sink ? 1u : 0u, s->qk_norm ? 1u : 0u, s->temp_every, s->softcap, s->temp_coef};
  return run_attention<true>(ma, a, s->cache_map, n_seq, rows, seq0, pos);
}

}  // extern "C"
