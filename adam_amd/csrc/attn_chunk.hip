// Softmax attention inside fixed chunks of the sequence, with a logarithmic distance penalty and no rotation.
//
// A token at position i sees positions floor(i / C) C .. i, so the cache of a sequence is one chunk per layer, token i at
// place i % C; what a new chunk overwrites is never seen again.  Values are cached divided by their root mean square.
//
// One token: k_chunk_attn_step, a workgroup per query head and span of SPAN keys; its own key and value come from the
// projections (the first query head of a key head stores them).  More than one span: k_chunk_attn_join.
//
// A portion of a prompt: k_chunk_attn_stage lays the keys the portion sees -- what the cache holds of the first token's
// chunk, then the portion's own -- out as matrix operands, K [np, dp] and V transposed [vp, np]; k_chunk_attn_keep then
// brings the cache up to date; k_chunk_attn_f32 / _bf16 take 16 queries of a head per wave through the keys of their
// chunks.  Scores arrive as K . Q^T, so a lane holds four keys of one query, which is also the layout the second
// product wants its right operand in: no shared memory.  float32: the float32 matrix instruction throughout.  bfloat16:
// keys and values rounded once, queries and softmax weights as sums of two bfloat16 terms, all sums in float32.
#include "linear_common.h"
#include <algorithm>

namespace adamah {

typedef AdamahChunkAttnSpec ASpec;
#define SPAN 512u
#define ATT_MASKED (-1.0e30f)

__device__ __forceinline__ float wsumf(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}
template <class T> __device__ __forceinline__ void load8(const T* p, float (&o)[8]);
template <> __device__ __forceinline__ void load8<float>(const float* p, float (&o)[8]) {
  const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
  o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w; o[4] = b.x; o[5] = b.y; o[6] = b.z; o[7] = b.w;
}
template <> __device__ __forceinline__ void load8<bf16_t>(const bf16_t* p, float (&o)[8]) {
  const uint4 a = *(const uint4*)p;
  o[0] = bf_lo(a.x); o[1] = bf_hi(a.x); o[2] = bf_lo(a.y); o[3] = bf_hi(a.y);
  o[4] = bf_lo(a.z); o[5] = bf_hi(a.z); o[6] = bf_lo(a.w); o[7] = bf_hi(a.w);
}

// ---- one token ------------------------------------------------------------------------------------------------------
// grid (heads, spans, sequences).  part: per (sequence, head, span) vdim + 2 floats {max, sum, values}, used when
// spans > 1.
template <class T>
__global__ void __launch_bounds__(256)
k_chunk_attn_step(const ASpec s, float* act, T* cache, float* part, uint32_t seq0, uint32_t pos) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float sh[12];
  const uint32_t D = s.dim, V = s.vdim, D8 = (D + 7u) & ~7u, V8 = (V + 7u) & ~7u, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
  const uint32_t h = blockIdx.x, row = blockIdx.z, rep = s.heads / s.kv_heads, kv = h / rep;
  const uint32_t n = pos % s.chunk + 1u, k0 = blockIdx.y * SPAN, k1 = min(n, k0 + SPAN);
  const bool own = k1 == n;                                     // this span ends with the token itself
  float *q = lds, *sc = q + D8, *vn = sc + SPAN, *red = vn + V8;  // red: [256 / (V8 / 8)][V8]
  const float* x = act + s.x + (uint64_t)row * s.x_stride;
  T* K = cache + (uint64_t)(seq0 + row) * s.seq_stride + s.k_off + (uint64_t)kv * s.chunk * D8;
  T* Vc = cache + (uint64_t)(seq0 + row) * s.seq_stride + s.v_off + (uint64_t)kv * s.chunk * V8;
  const float* xk = x + s.x_k + kv * D;
  const float* xv = x + s.x_v + kv * V;
  float qk = 0.f, vv = 0.f;
  for (uint32_t d = tid; d < D8; d += 256u) {
    const float t = d < D ? x[s.x_q + h * D + d] : 0.f;
    q[d] = t;
    if (d < D) qk = fmaf(t, xk[d], qk);
  }
  for (uint32_t d = tid; d < V; d += 256u) vv = fmaf(xv[d], xv[d], vv);
  qk = wsumf(qk); vv = wsumf(vv);
  if (lane == 0) { sh[wave] = qk; sh[4 + wave] = vv; }
  __syncthreads();
  qk = (sh[0] + sh[1]) + (sh[2] + sh[3]);
  const float iv = 1.0f / sqrtf(((sh[4] + sh[5]) + (sh[6] + sh[7])) / (float)V + s.eps);
  const float r1 = act[s.r1 + h], r2 = act[s.r2 + h];
  for (uint32_t d = tid; d < V8; d += 256u) vn[d] = d < V ? xv[d] * iv : 0.f;
  if (own && h % rep == 0) {
    for (uint32_t d = tid; d < D8; d += 256u) K[(uint64_t)(n - 1u) * D8 + d] = (T)(d < D ? xk[d] : 0.f);
    for (uint32_t d = tid; d < V8; d += 256u) Vc[(uint64_t)(n - 1u) * V8 + d] = (T)(d < V ? xv[d] * iv : 0.f);
  }
  // scores: 16 lanes a key
  const uint32_t l16 = lane & 15u, kq = lane >> 4, last = own ? k1 - 1u : k1;   // cached keys of the span: [k0, last)
  for (uint32_t j = k0 + wave * 4u; j < last; j += 16u) {
    const uint32_t key = j + kq;
    float a = 0.f;
    if (key < last)
      for (uint32_t c = l16 * 8u; c < D8; c += 128u) {
        float kk[8];
        load8<T>(K + (uint64_t)key * D8 + c, kk);
#pragma unroll
        for (int i = 0; i < 8; i++) a = fmaf(kk[i], q[c + i], a);
      }
    a += __shfl_xor(a, 1, 64); a += __shfl_xor(a, 2, 64); a += __shfl_xor(a, 4, 64); a += __shfl_xor(a, 8, 64);
    if (l16 == 0 && key < last) sc[key - k0] = a * s.scale - r1 * log1pf(r2 * (float)(n - 1u - key));
  }
  if (own && tid == 0) sc[k1 - 1u - k0] = qk * s.scale;          // distance 0: ln 1 = 0
  __syncthreads();
  float mx = ATT_MASKED, sum = 0.f;
  for (uint32_t j = tid; j < k1 - k0; j += 256u) mx = fmaxf(mx, sc[j]);
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
  if (lane == 0) sh[wave] = mx;
  __syncthreads();
  mx = fmaxf(fmaxf(sh[0], sh[1]), fmaxf(sh[2], sh[3]));
  for (uint32_t j = tid; j < k1 - k0; j += 256u) { const float e = expf(sc[j] - mx); sc[j] = e; sum += e; }
  sum = wsumf(sum);
  if (lane == 0) sh[8 + wave] = sum;
  __syncthreads();
  sum = (sh[8] + sh[9]) + (sh[10] + sh[11]);
  // values: 8 columns a thread, keys dealt out over the thread groups
  const uint32_t nc = V8 >> 3, ng = 256u / nc, gi = tid / nc, c8 = (tid - gi * nc) * 8u;
  float o[8] = {0, 0, 0, 0, 0, 0, 0, 0};
  if (gi < ng) {
    for (uint32_t key = k0 + gi; key < last; key += ng) {
      float t[8];
      load8<T>(Vc + (uint64_t)key * V8 + c8, t);
      const float p = sc[key - k0];
#pragma unroll
      for (int i = 0; i < 8; i++) o[i] = fmaf(p, t[i], o[i]);
    }
#pragma unroll
    for (int i = 0; i < 8; i++) red[gi * V8 + c8 + i] = o[i];
  }
  __syncthreads();
  const float pw = own ? sc[k1 - 1u - k0] : 0.f;
  for (uint32_t d = tid; d < V; d += 256u) {
    float a = pw * vn[d];
    for (uint32_t gg = 0; gg < ng; gg++) a += red[gg * V8 + d];
    if (gridDim.y == 1) act[s.out + (uint64_t)row * s.out_stride + h * V + d] = a / sum;
    else part[(((uint64_t)row * s.heads + h) * gridDim.y + blockIdx.y) * (V + 2u) + 2u + d] = a;
  }
  if (gridDim.y > 1 && tid == 0) {
    float* p = part + (((uint64_t)row * s.heads + h) * gridDim.y + blockIdx.y) * (V + 2u);
    p[0] = mx; p[1] = sum;
  }
}
__global__ void __launch_bounds__(128)
k_chunk_attn_join(const ASpec s, float* act, const float* __restrict__ part, uint32_t n_part) {
  const uint32_t h = blockIdx.x, row = blockIdx.y, V = s.vdim;
  const float* p = part + ((uint64_t)row * s.heads + h) * n_part * (V + 2u);
  float mx = ATT_MASKED, sum = 0.f;
  for (uint32_t i = 0; i < n_part; i++) mx = fmaxf(mx, p[(uint64_t)i * (V + 2u)]);
  for (uint32_t i = 0; i < n_part; i++) sum += p[(uint64_t)i * (V + 2u) + 1u] * expf(p[(uint64_t)i * (V + 2u)] - mx);
  for (uint32_t d = threadIdx.x; d < V; d += 128u) {
    float a = 0.f;
    for (uint32_t i = 0; i < n_part; i++) a = fmaf(expf(p[(uint64_t)i * (V + 2u)] - mx), p[(uint64_t)i * (V + 2u) + 2u + d], a);
    act[s.out + (uint64_t)row * s.out_stride + h * V + d] = a / sum;
  }
}

// ---- a portion ------------------------------------------------------------------------------------------------------
struct StageDims { uint32_t past, n, np, dp, vp; };   // keys from the cache, keys in all, padded counts
// One workgroup per 32 staged keys and key head.  K: [kv_heads, np, dp], VT: [kv_heads, vp, np].
template <class T>
__global__ void __launch_bounds__(256)
k_chunk_attn_stage(const ASpec s, const float* __restrict__ act, const T* cache, T* __restrict__ K, T* __restrict__ VT, StageDims sd) {
  extern __shared__ float vt[];                    // [32][V + 1]
  __shared__ float inv[32];
  const uint32_t D = s.dim, V = s.vdim, D8 = (D + 7u) & ~7u, V8 = (V + 7u) & ~7u, tid = threadIdx.x, kv = blockIdx.y, j0 = blockIdx.x * 32u;
  const T* cK = cache + s.k_off + (uint64_t)kv * s.chunk * D8;
  const T* cV = cache + s.v_off + (uint64_t)kv * s.chunk * V8;
  const float* xk = act + s.x + s.x_k + kv * D;
  const float* xv = act + s.x + s.x_v + kv * V;
  {                                                // root mean squares of the new values: 8 threads a key
    const uint32_t j = j0 + (tid >> 3);
    float ss = 0.f;
    if (j >= sd.past && j < sd.n)
      for (uint32_t d = tid & 7u; d < V; d += 8u) { const float v = xv[(uint64_t)(j - sd.past) * s.x_stride + d]; ss = fmaf(v, v, ss); }
    ss += __shfl_xor(ss, 1, 64); ss += __shfl_xor(ss, 2, 64); ss += __shfl_xor(ss, 4, 64);
    if ((tid & 7u) == 0) inv[tid >> 3] = 1.0f / sqrtf(ss / (float)V + s.eps);
  }
  __syncthreads();
  for (uint32_t i = tid; i < 32u * sd.dp; i += 256u) {
    const uint32_t jj = i / sd.dp, d = i - jj * sd.dp, j = j0 + jj;
    T v = (T)0.f;
    if (d < D && j < sd.n) v = j < sd.past ? cK[(uint64_t)j * D8 + d] : (T)xk[(uint64_t)(j - sd.past) * s.x_stride + d];
    K[((uint64_t)kv * sd.np + j) * sd.dp + d] = v;
  }
  for (uint32_t i = tid; i < 32u * V; i += 256u) {
    const uint32_t jj = i / V, d = i - jj * V, j = j0 + jj;
    float v = 0.f;
    if (j < sd.n) v = j < sd.past ? (float)cV[(uint64_t)j * V8 + d] : xv[(uint64_t)(j - sd.past) * s.x_stride + d] * inv[jj];
    vt[jj * (V + 1u) + d] = v;
  }
  __syncthreads();
  for (uint32_t i = tid; i < 32u * sd.vp; i += 256u) {
    const uint32_t d = i >> 5, jj = i & 31u;
    VT[((uint64_t)kv * sd.vp + d) * sd.np + j0 + jj] = (T)(d < V ? vt[jj * (V + 1u) + d] : 0.f);
  }
}
// The cache after the portion: the tokens of the last token's chunk.  A launch of its own, behind the staging that
// still reads the places it writes.
template <class T>
__global__ void __launch_bounds__(256)
k_chunk_attn_keep(const ASpec s, T* cache, const T* __restrict__ K, const T* __restrict__ VT, StageDims sd, uint32_t first, uint32_t place) {
  const uint32_t D8 = (s.dim + 7u) & ~7u, V8 = (s.vdim + 7u) & ~7u, kv = blockIdx.y, j = first + blockIdx.x;
  T* cK = cache + s.k_off + ((uint64_t)kv * s.chunk + place + blockIdx.x) * D8;
  T* cV = cache + s.v_off + ((uint64_t)kv * s.chunk + place + blockIdx.x) * V8;
  for (uint32_t d = threadIdx.x; d < D8; d += 256u) cK[d] = K[((uint64_t)kv * sd.np + j) * sd.dp + d];
  for (uint32_t d = threadIdx.x; d < V8; d += 256u) cV[d] = VT[((uint64_t)kv * sd.vp + d) * sd.np + j];
}

// 16 queries of a head per wave.  float32 form: keys 16 at a time.
template <int NV>
__global__ void __launch_bounds__(256)
k_chunk_attn_f32(const ASpec s, float* act, const float* __restrict__ K, const float* __restrict__ VT, StageDims sd, uint32_t m, uint32_t pos) {
  const uint32_t lane = threadIdx.x & 63u, c = lane & 15u, kg = lane >> 4, h = blockIdx.x, kv = h / (s.heads / s.kv_heads);
  const uint32_t q0 = (blockIdx.y * 4u + (threadIdx.x >> 6)) * 16u;
  if (q0 >= m) return;
  const uint32_t qr = min(q0 + c, m - 1u), base = pos - sd.past;           // key j of the stage sits at position base + j
  const uint32_t qj = sd.past + qr, lo = (pos + qr) / s.chunk * s.chunk - base;   // visible: lo .. qj
  const uint32_t first = ((pos + q0) / s.chunk * s.chunk - base) & ~15u, end = sd.past + min(q0 + 16u, m);
  const float* xq = act + s.x + (uint64_t)qr * s.x_stride + s.x_q + h * s.dim;
  const float* kb = K + (uint64_t)kv * sd.np * sd.dp;
  const float* vb = VT + (uint64_t)kv * sd.vp * sd.np;
  const float r1 = act[s.r1 + h], r2 = act[s.r2 + h];
  f4_t o[NV];
#pragma unroll
  for (int i = 0; i < NV; i++) o[i] = (f4_t){0, 0, 0, 0};
  float mx = ATT_MASKED, sum = 0.f;
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

// bfloat16 form: keys 32 at a time (two tiles of 16); DK: k-steps of 32 dimensions.
template <int DK, int NV>
__global__ void __launch_bounds__(256)
k_chunk_attn_bf16(const ASpec s, float* act, const bf16_t* __restrict__ K, const bf16_t* __restrict__ VT, StageDims sd, uint32_t m, uint32_t pos) {
  const uint32_t lane = threadIdx.x & 63u, c = lane & 15u, kg = lane >> 4, h = blockIdx.x, kv = h / (s.heads / s.kv_heads);
  const uint32_t q0 = (blockIdx.y * 4u + (threadIdx.x >> 6)) * 16u;
  if (q0 >= m) return;
  const uint32_t qr = min(q0 + c, m - 1u), base = pos - sd.past;
  const uint32_t qj = sd.past + qr, lo = (pos + qr) / s.chunk * s.chunk - base;
  const uint32_t first = ((pos + q0) / s.chunk * s.chunk - base) & ~31u, end = sd.past + min(q0 + 16u, m);
  const uint32_t lo_all = (pos + min(q0 + 15u, m - 1u)) / s.chunk * s.chunk - base;    // seen by every query from here ..
  const float* xq = act + s.x + (uint64_t)qr * s.x_stride + s.x_q + h * s.dim;
  const bf16_t* kb = K + (uint64_t)kv * sd.np * sd.dp;
  const bf16_t* vb = VT + (uint64_t)kv * sd.vp * sd.np;
  const float r1 = act[s.r1 + h], r2 = act[s.r2 + h];
  bf8_t qh[DK], ql[DK];
#pragma unroll
  for (int t = 0; t < DK; t++)
#pragma unroll
    for (int i = 0; i < 8; i++) {
      const uint32_t d = 32u * t + 8u * kg + i;
      const float x = d < s.dim ? xq[d] * s.scale : 0.f;
      qh[t][i] = (bf16_t)x;
      ql[t][i] = (bf16_t)(x - (float)qh[t][i]);
    }
  f4_t o[NV];
#pragma unroll
  for (int i = 0; i < NV; i++) o[i] = (f4_t){0, 0, 0, 0};
  float mx = ATT_MASKED, sum = 0.f;
  for (uint32_t j0 = first; j0 < end; j0 += 32u) {
    f4_t a[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}};
#pragma unroll
    for (int t = 0; t < DK; t++)
#pragma unroll
      for (int u = 0; u < 2; u++) {
        const bf8_t kk = *(const bf8_t*)(kb + (uint64_t)(j0 + 16u * u + c) * sd.dp + 32u * t + 8u * kg);
        a[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kk, ql[t], a[u], 0, 0, 0);
        a[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kk, qh[t], a[u], 0, 0, 0);
      }
    const bool all = j0 >= lo_all && j0 + 31u <= sd.past + q0;             // .. to here
    float t = ATT_MASKED;
#pragma unroll
    for (int u = 0; u < 2; u++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const uint32_t j = j0 + 16u * u + 4u * kg + i;
        const bool ok = all || (j >= lo && j <= qj);
        a[u][i] = ok ? a[u][i] - r1 * __logf(fmaf(r2, (float)(qj - j), 1.0f)) : ATT_MASKED;
        t = fmaxf(t, a[u][i]);
      }
    t = fmaxf(t, __shfl_xor(t, 16, 64)); t = fmaxf(t, __shfl_xor(t, 32, 64));
    const float nm = fmaxf(mx, t), al = __expf(mx - nm);
    mx = nm;
    float ps = 0.f;
    bf8_t ph, pl;
#pragma unroll
    for (int u = 0; u < 2; u++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const float p = a[u][i] > 0.5f * ATT_MASKED ? __expf(a[u][i] - nm) : 0.f;
        ps += p;
        ph[4 * u + i] = (bf16_t)p;
        pl[4 * u + i] = (bf16_t)(p - (float)ph[4 * u + i]);
      }
    ps += __shfl_xor(ps, 16, 64); ps += __shfl_xor(ps, 32, 64);
    sum = fmaf(sum, al, ps);
#pragma unroll
    for (int v = 0; v < NV; v++) {
      const bf16_t* src = vb + (uint64_t)(v * 16u + c) * sd.np + j0 + 4u * kg;
      const bf4_t v0 = *(const bf4_t*)src, v1 = *(const bf4_t*)(src + 16);
      const bf8_t vv = {v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
      o[v] *= al;
      o[v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vv, pl, o[v], 0, 0, 0);
      o[v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vv, ph, o[v], 0, 0, 0);
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

static Scratch g_stage, g_parts;
void attn_chunk_release() { scratch_free(g_stage); scratch_free(g_parts); }

template <int DK>
static void launch_bf16(const ASpec& s, float* act, const bf16_t* K, const bf16_t* VT, const StageDims& sd, uint32_t m, uint32_t pos) {
  const dim3 grid(s.heads, cdiv(m, 64));
  switch (sd.vp / 16u) {
#define CASE(N) case N: k_chunk_attn_bf16<DK, N><<<grid, 256, 0, g.stream>>>(s, act, K, VT, sd, m, pos); break
    CASE(2); CASE(4); CASE(6); CASE(8); CASE(12); CASE(16);
#undef CASE
  }
}
static uint32_t vtiles(uint32_t v) {
  for (uint32_t t : {2u, 4u, 6u, 8u, 12u, 16u}) if (v <= 16u * t) return t;
  return 0;
}

template <class T>
static int run_portion(const ASpec& s, float* act, T* cache, uint32_t m, uint32_t pos) {
  StageDims sd;
  sd.past = pos % s.chunk;
  sd.n = sd.past + m;
  sd.np = (sd.n + 31u) & ~31u;
  sd.dp = 32u * (s.dim <= 128u ? cdiv(s.dim, 32) : s.dim <= 192u ? 6u : 8u);
  sd.vp = vtiles(s.vdim) * 16u;
  const uint64_t nk = (uint64_t)s.kv_heads * sd.np * sd.dp, nv = (uint64_t)s.kv_heads * sd.np * sd.vp;
  if (int r = scratch_need(g_stage, (nk + nv) * sizeof(T) + 64)) return r;
  T *K = (T*)g_stage.p, *VT = K + nk;
  k_chunk_attn_stage<T><<<dim3(sd.np / 32u, s.kv_heads), 256, (size_t)32 * (s.vdim + 1) * 4, g.stream>>>(s, act, cache, K, VT, sd);
  count_launch();
  if (int r = check_launch()) return r;
  // positions still wanted after the portion: the last token's chunk, from its first new token on
  const uint32_t end = pos + m, chunk0 = (end - 1u) / s.chunk * s.chunk, from = std::max(chunk0, pos);
  k_chunk_attn_keep<T><<<dim3(end - from, s.kv_heads), 256, 0, g.stream>>>(s, cache, K, VT, sd, from - (pos - sd.past), from % s.chunk);
  count_launch();
  if (int r = check_launch()) return r;
  if constexpr (sizeof(T) == 4) {
    const dim3 grid(s.heads, cdiv(m, 64));
    if (sd.vp <= 64u) k_chunk_attn_f32<4><<<grid, 256, 0, g.stream>>>(s, act, K, VT, sd, m, pos);
    else k_chunk_attn_f32<16><<<grid, 256, 0, g.stream>>>(s, act, K, VT, sd, m, pos);
  } else {
    switch (sd.dp / 32u) {
      case 1: launch_bf16<1>(s, act, K, VT, sd, m, pos); break;
      case 2: launch_bf16<2>(s, act, K, VT, sd, m, pos); break;
      case 3: launch_bf16<3>(s, act, K, VT, sd, m, pos); break;
      case 4: launch_bf16<4>(s, act, K, VT, sd, m, pos); break;
      case 6: launch_bf16<6>(s, act, K, VT, sd, m, pos); break;
      default: launch_bf16<8>(s, act, K, VT, sd, m, pos); break;
    }
  }
  count_launch();
  return check_launch();
}

template <class T>
static int run_step(const ASpec& s, float* act, T* cache, uint32_t n_seq, uint32_t seq0, uint32_t pos) {
  const uint32_t spans = cdiv(pos % s.chunk + 1u, SPAN), V8 = (s.vdim + 7u) & ~7u, D8 = (s.dim + 7u) & ~7u;
  if (s.chunk > SPAN)      // at its full size from the first step on: a graph may be recording when the second span begins
    if (int r = scratch_need(g_parts, (size_t)n_seq * s.heads * cdiv(s.chunk, SPAN) * (s.vdim + 2) * 4)) return r;
  const size_t lds = ((size_t)D8 + SPAN + V8 + (256 / (V8 / 8)) * V8) * 4;
  k_chunk_attn_step<T><<<dim3(s.heads, spans, n_seq), 256, lds, g.stream>>>(s, act, cache, (float*)g_parts.p, seq0, pos);
  count_launch();
  if (spans > 1) {
    if (int r = check_launch()) return r;
    k_chunk_attn_join<<<dim3(s.heads, n_seq), 128, 0, g.stream>>>(s, act, (const float*)g_parts.p, spans);
    count_launch();
  }
  return check_launch();
}

}  // namespace adamah

using namespace adamah;

extern "C" int adamah_chunk_attention_dev(uint32_t map_act, uint32_t h_spec, uint32_t n_seq, uint32_t rows, uint32_t seq0, uint32_t pos) { ADAMAH_API();
  Map* ma = get_f32_map(map_act);
  const ASpec* s = spec_of<ASpec>(h_spec);
  if (!ma || !s || n_seq == 0 || rows == 0 || (n_seq > 1 && rows > 1)) return ADAMAH_ERR_INVALID;
  Map* mc = get_map(s->cache_map);
  if (!mc || (mc->dtype != DTYPE_F32 && mc->dtype != DTYPE_BF16)) return ADAMAH_ERR_INVALID;
  const uint64_t D = s->dim, V = s->vdim, H = s->heads, G = s->kv_heads, C = s->chunk, n_tok = (uint64_t)n_seq * rows;
  const uint64_t D8 = (D + 7) / 8 * 8, V8 = (V + 7) / 8 * 8;
  if (D == 0 || D > 256 || V == 0 || V > 256 || H == 0 || G == 0 || H % G || C == 0 || (uint64_t)pos + rows > 0xFFFFFF00ull) return ADAMAH_ERR_INVALID;
  if (s->x_q + H * D > s->x_stride || s->x_k + G * D > s->x_stride || s->x_v + G * V > s->x_stride ||
      !in_range(s->x, (n_tok - 1) * s->x_stride + s->x_stride, ma->n_elems) ||
      !in_range(s->out, (n_tok - 1) * s->out_stride + H * V, ma->n_elems) ||
      !in_range(s->r1, H, ma->n_elems) || !in_range(s->r2, H, ma->n_elems)) return ADAMAH_ERR_INVALID;
  if (((s->k_off | s->v_off | s->seq_stride) & 7u) || s->k_off + G * C * D8 > s->seq_stride || s->v_off + G * C * V8 > s->seq_stride ||
      !in_range((uint64_t)seq0 * s->seq_stride, (uint64_t)n_seq * s->seq_stride, mc->n_elems)) return ADAMAH_ERR_INVALID;
  float* act = (float*)ma->buf;
  const uint64_t slot = (uint64_t)seq0 * s->seq_stride;
  if (rows == 1)
    return mc->dtype == DTYPE_F32 ? run_step<float>(*s, act, (float*)mc->buf, n_seq, seq0, pos) : run_step<bf16_t>(*s, act, (bf16_t*)mc->buf, n_seq, seq0, pos);
  return mc->dtype == DTYPE_F32 ? run_portion<float>(*s, act, (float*)mc->buf + slot, rows, pos)
                                : run_portion<bf16_t>(*s, act, (bf16_t*)mc->buf + slot, rows, pos);
}
