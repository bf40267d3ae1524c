// Sequence mixers that carry a matrix state per head: the gated delta rule with a decay per key channel, and retention
// (one fixed decay per head).  State, decays, step sizes, unit norms and the products with the state are float32.
//
// One token (decode): k_delta_step / k_retention_step.  A workgroup owns one head and 32 of its value columns; the
// state's columns are independent but for the vectors every workgroup of a head makes for itself (convolution, unit
// norms, decay), so no workgroup waits for another.
//
// A portion of a prompt: two launches.  The first (k_delta_prep / k_retention_prep, a workgroup per head and chunk of
// 16 tokens, all chunks at once) writes what a chunk does to the state as dense operands; the second (k_chunk_scan, a
// workgroup per head and 16 value columns) walks over the chunks with the state in the accumulators of the float32
// matrix instruction.  With b_t the step size, G_t the product of the decays up to token t of the chunk and S the state
// ahead of it:
//   A[t,s] = sum_d k_t k_s G_t / G_s  (s < t),   T = (I + diag(b) A)^-1,   U = T diag(b) (V - (G k) S)
//   o_t = S^T (G_t q_t) + sum_{s <= t} B[t,s] u_s,   B[t,s] = sum_d q_t k_s G_t / G_s
//   S  <- G_last S + sum_s (G_last / G_s) k_s u_s^T
// (retention: U = V).  Decays are kept as logarithms and every quotient is the exponential of a difference that is <= 0,
// so a decay as strong as float32 can hold neither overflows nor loses the tokens behind it.
#include "recurrent_common.h"
#include <algorithm>

namespace adamah {


typedef AdamahDeltaSpec DSpec;
typedef AdamahRetentionSpec RSpec;

// sums over a workgroup of NW waves of up to three values at once; sh: 3 NW floats
template <int NW>
__device__ __forceinline__ void block_add3(float& a, float& b, float& c, float* sh) {
  a = wave_add(a); b = wave_add(b); c = wave_add(c);
  const uint32_t w = threadIdx.x >> 6;
  __syncthreads();
  if ((threadIdx.x & 63u) == 0) { sh[w] = a; sh[NW + w] = b; sh[2 * NW + w] = c; }
  __syncthreads();
  a = b = c = 0.f;
#pragma unroll
  for (int i = 0; i < NW; i++) { a += sh[i]; b += sh[NW + i]; c += sh[2 * NW + i]; }
}

// dot product of a bf16 matrix row of kp columns (a multiple of 64, zeros at the end) with a float32 vector of as many,
// by 8 neighbouring lanes (all get the sum)
__device__ __forceinline__ float dot8(const bf16_t* w, const float* x, uint32_t kp, uint32_t sub) {
  float a = 0.f;
  for (uint32_t c = sub * 8u; c < kp; c += 64u) {
    const uint4 p = *(const uint4*)(w + c);
    const uint32_t u[4] = {p.x, p.y, p.z, p.w};
#pragma unroll
    for (int i = 0; i < 4; i++) { a = fmaf(bf_lo(u[i]), x[c + 2 * i], a); a = fmaf(bf_hi(u[i]), x[c + 2 * i + 1], a); }
  }
  a += __shfl_xor(a, 1, 64); a += __shfl_xor(a, 2, 64); a += __shfl_xor(a, 4, 64);
  return a;
}

struct LowRank { uint32_t w, k, k_stride, src, src_stride, out, out_stride; };   // what a step needs of a linear spec

// the same for a row held in registers: NC 16-byte words of it per lane (zeros beyond the row), x as long
template <int NC>
__device__ __forceinline__ float dot8_regs(const uint4 (&w)[NC], const float* x, uint32_t kp, uint32_t sub) {
  float a = 0.f;
#pragma unroll
  for (int n = 0; n < NC; n++) {
    const uint32_t c = sub * 8u + 64u * n, u[4] = {w[n].x, w[n].y, w[n].z, w[n].w};
    if (c >= kp) break;
#pragma unroll
    for (int i = 0; i < 4; i++) { a = fmaf(bf_lo(u[i]), x[c + 2 * i], a); a = fmaf(bf_hi(u[i]), x[c + 2 * i + 1], a); }
  }
  a += __shfl_xor(a, 1, 64); a += __shfl_xor(a, 2, 64); a += __shfl_xor(a, 4, 64);
  return a;
}

// One token of one sequence per blockIdx.z; DN: state rows a thread holds (dim <= 16 DN); TM >= taps.  Everything a
// workgroup reads is asked for at the start: the state, the convolution's inputs, the rows of the low-rank factors (in
// registers where their rank is at most 128).
#define DSTEP 512u
template <int DN, int TM>
__global__ void __launch_bounds__(DSTEP)
k_delta_step(const DSpec s, const LowRank da, const LowRank ga, float* act, const bf16_t* __restrict__ W, float* state, uint32_t seq0,
             uint32_t pos) {
  constexpr int NP = DN / 4 > 0 ? DN / 4 : 1;          // decay rows of 8 lanes: 64 a pass
  constexpr uint32_t NG = DSTEP / VC;
  extern __shared__ float lds[];
  __shared__ float sh[3 * DSTEP / 64];
  __shared__ float red[2][NG][VC];
  __shared__ float vs[VC];
  const uint32_t D = s.dim, V = s.vdim, tid = threadIdx.x, h = blockIdx.x, v0 = blockIdx.y * VC, row = blockIdx.z;
  float *qs = lds, *ks = qs + D, *gs = ks + D, *la = gs + D, *lg = la + da.k_stride;
  const uint32_t n_ch = 2u * s.kv_heads * D + s.heads * V, rep = s.heads / s.kv_heads, kv = h / rep, sub = tid & 7u;
  const float* x = act + s.x + (uint64_t)row * s.x_stride;
  float* ring = state + (uint64_t)(seq0 + row) * s.seq_stride + s.conv_off;
  float* S = state + (uint64_t)(seq0 + row) * s.seq_stride + s.s_off + (uint64_t)h * D * V;
  const uint32_t qc = kv * D, kc = s.kv_heads * D + kv * D, vc = 2u * s.kv_heads * D + h * V;
  const uint32_t col = tid & (VC - 1u), dg = tid / VC, v = v0 + col;
  const bool small = da.k_stride <= 128u && ga.k_stride <= 128u;
  const uint32_t gt = DSTEP - 1u - tid, gv = v0 + (gt >> 3), grow = h * V + min(gv, V - 1u);   // gate rows: the last threads
  float st[DN];
#pragma unroll
  for (int i = 0; i < DN; i++) {
    const uint32_t d = dg + NG * i;
    st[i] = (pos != 0u && d < D && v < V) ? S[(uint64_t)d * V + v] : 0.f;
  }
  for (uint32_t i = tid; i < da.k_stride; i += DSTEP) la[i] = i < da.k ? act[da.src + (uint64_t)row * da.src_stride + i] : 0.f;
  for (uint32_t i = gt; i < ga.k_stride; i += DSTEP) lg[i] = i < ga.k ? act[ga.src + (uint64_t)row * ga.src_stride + i] : 0.f;
  uint4 wa[NP][2], wg[2];
  float bias[NP];
#pragma unroll
  for (int i = 0; i < NP; i++) {
    const uint32_t r = h * D + min((tid >> 3) + 64u * i, D - 1u);
    bias[i] = act[s.dt_bias + r];
    if (small)
#pragma unroll
      for (int n = 0; n < 2; n++)
        wa[i][n] = sub * 8u + 64u * n < da.k_stride ? *(const uint4*)(W + da.w + (uint64_t)r * da.k_stride + sub * 8u + 64u * n) : make_uint4(0, 0, 0, 0);
  }
  const float a_log = act[s.a_log + h], step = x[s.x_b + h];
  if (small && gt < 8u * VC)
#pragma unroll
    for (int n = 0; n < 2; n++)
      wg[n] = (gt & 7u) * 8u + 64u * n < ga.k_stride ? *(const uint4*)(W + ga.w + (uint64_t)grow * ga.k_stride + (gt & 7u) * 8u + 64u * n) : make_uint4(0, 0, 0, 0);
  float sq = 0.f, sk = 0.f, qk = 0.f;
  for (uint32_t i = tid; i < 2u * D; i += DSTEP) {
    const bool is_k = i >= D;
    const uint32_t d = is_k ? i - D : i;
    const float a = conv_silu_ring<TM>(x, ring, n_ch, (is_k ? kc : qc) + d, pos, act + (is_k ? s.ck : s.cq) + (uint64_t)(kv * D + d) * s.taps, s.taps);
    (is_k ? ks : qs)[d] = a;
    if (is_k) sk = fmaf(a, a, sk); else sq = fmaf(a, a, sq);
  }
  if (gt < VC && v0 + gt < V)
    vs[gt] = conv_silu_ring<TM>(x, ring, n_ch, vc + v0 + gt, pos, act + s.cv + (uint64_t)(h * V + v0 + gt) * s.taps, s.taps);
  const float ea = expf(a_log), beta = sigmoid_f(step);
  __syncthreads();
  for (uint32_t d = tid; d < D; d += DSTEP) qk = fmaf(qs[d], ks[d], qk);
  if (small) {
#pragma unroll
    for (int i = 0; i < NP; i++) {
      const uint32_t d = (tid >> 3) + 64u * i;
      const float a = dot8_regs<2>(wa[i], la, da.k_stride, sub);
      if (sub == 0 && d < D) gs[d] = expf(-ea * softplus_f(a + bias[i]));
    }
  } else {
    for (uint32_t d = tid >> 3; d < ((D + 63u) & ~63u); d += 64u) {      // whole waves take part in the dot products
      const uint32_t r = h * D + min(d, D - 1u);
      const float a = dot8(W + da.w + (uint64_t)r * da.k_stride, la, da.k_stride, sub);
      if (sub == 0 && d < D) gs[d] = expf(-ea * softplus_f(a + act[s.dt_bias + r]));
    }
  }
  if (gt < 8u * VC) {
    const float a = small ? dot8_regs<2>(wg, lg, ga.k_stride, gt & 7u) : dot8(W + ga.w + (uint64_t)grow * ga.k_stride, lg, ga.k_stride, gt & 7u);
    if ((gt & 7u) == 0 && gv < V) act[ga.out + (uint64_t)row * ga.out_stride + grow] = a;
  }
  block_add3<DSTEP / 64>(sq, sk, qk, sh);      // (its barriers also publish gs)
  const float iq = 1.0f / sqrtf(sq + 1e-6f) / sqrtf((float)D), ik = 1.0f / sqrtf(sk + 1e-6f);
  qk = qk * iq * ik;
  float pk = 0.f, pq = 0.f;
#pragma unroll
  for (int i = 0; i < DN; i++) {
    const uint32_t d = dg + NG * i;
    if (d < D) {
      st[i] *= gs[d];
      pk = fmaf(st[i], ks[d], pk); pq = fmaf(st[i], qs[d], pq);
    }
  }
  red[0][dg][col] = pk; red[1][dg][col] = pq;
  __syncthreads();
  pk = 0.f; pq = 0.f;
#pragma unroll
  for (int i = 0; i < (int)NG; i++) { pk += red[0][i][col]; pq += red[1][i][col]; }
  if (v < V) {
    const float u = beta * (vs[col] - pk * ik);
    if (dg == 0) act[s.out + (uint64_t)row * s.out_stride + h * V + v] = fmaf(u, qk, pq * iq);
    const float uk = u * ik;
#pragma unroll
    for (int i = 0; i < DN; i++) {
      const uint32_t d = dg + NG * i;
      if (d < D) S[(uint64_t)d * V + v] = fmaf(ks[d], uk, st[i]);
    }
  }
  float* slot = ring + (uint64_t)(pos % s.taps) * n_ch;
  if (blockIdx.y == 0 && h % rep == 0)
    for (uint32_t d = tid; d < D; d += DSTEP) { slot[qc + d] = x[qc + d]; slot[kc + d] = x[kc + d]; }
  if (tid < VC && v0 + tid < V) slot[vc + v0 + tid] = x[vc + v0 + tid];
}

__device__ __forceinline__ float rotated(const float* x, const float* freq, uint32_t d, uint32_t dims, uint32_t p) {
  const uint32_t half = dims >> 1;
  if (d >= dims) return x[d];
  const uint32_t i = d < half ? d : d - half;
  float sn, cs;
  sincosf((float)p * freq[i], &sn, &cs);
  return d < half ? x[d] * cs - x[d + half] * sn : x[d] * cs + x[d - half] * sn;
}

template <int DN>
__global__ void __launch_bounds__(256)
k_retention_step(const RSpec s, float* act, float* state, uint32_t seq0, uint32_t pos) {
  extern __shared__ float lds[];
  __shared__ float sh[12];
  __shared__ float red[8][VC];
  const uint32_t D = s.dim, V = s.vdim, tid = threadIdx.x, h = blockIdx.x, v0 = blockIdx.y * VC, row = blockIdx.z;
  float *qs = lds, *ks = qs + D;
  const float* x = act + s.x + (uint64_t)row * s.x_stride;
  float* S = state + (uint64_t)(seq0 + row) * s.seq_stride + s.s_off + (uint64_t)h * D * V;
  const uint32_t col = tid & 31u, dg = tid >> 5, v = v0 + col;
  const float dec = act[s.decay + h], kscale = 1.0f / sqrtf((float)D);
  float st[DN];
#pragma unroll
  for (int i = 0; i < DN; i++) {
    const uint32_t d = dg + 8u * i;
    st[i] = (pos != 0u && d < D && v < V) ? S[(uint64_t)d * V + v] : 0.f;
  }
  const float vv = v < V ? x[s.x_v + h * V + v] : 0.f;
  float qk = 0.f, z0 = 0.f, z1 = 0.f;
  for (uint32_t d = tid; d < D; d += 256u) {
    qs[d] = rotated(x + s.x_q + h * D, act + s.freq, d, s.rot_dims, pos);
    ks[d] = rotated(x + s.x_k + h * D, act + s.freq, d, s.rot_dims, pos) * kscale;
    qk = fmaf(qs[d], ks[d], qk);
  }
  block_add3<4>(qk, z0, z1, sh);
  float pq = 0.f;
#pragma unroll
  for (int i = 0; i < DN; i++) {
    const uint32_t d = dg + 8u * i;
    if (d < D && v < V) {
      const float t = dec * st[i];
      pq = fmaf(t, qs[d], pq);
      S[(uint64_t)d * V + v] = fmaf(ks[d], vv, t);
    }
  }
  red[dg][col] = pq;
  __syncthreads();
  if (dg == 0 && v < V) {
    pq = 0.f;
#pragma unroll
    for (int i = 0; i < 8; i++) pq += red[i][col];
    act[s.out + (uint64_t)row * s.out_stride + h * V + v] = fmaf(vv, qk, pq);
  }
}

// ---- chunk operands -------------------------------------------------------------------------------------------------
// Block of one (head, chunk): W = T diag(b) (G k) [16][Dp], Q = G q [16][Dp], K^T [Dp][16], B [16][16], U0 [16][Vp], G_last [Dp].
struct ChunkDims { uint32_t Dp, Vp, n_chunks; };
__host__ __device__ inline uint32_t chunk_floats(uint32_t Dp, uint32_t Vp) { return 49u * Dp + 256u + 16u * Vp; }

// Columns of q and k (a thread each) run through their convolution in registers, then those of v and of the decay.
template <int TM>
__global__ void __launch_bounds__(256)
k_delta_prep(const DSpec s, uint32_t dec_out, uint32_t dec_stride, const float* __restrict__ act, const float* __restrict__ state,
             float* __restrict__ scratch, ChunkDims cd, uint32_t m, uint32_t seq0, uint32_t pos) {
  extern __shared__ float lds[];
  __shared__ __attribute__((aligned(16))) float A[CH][CH + 4], M[CH][CH + 4];
  __shared__ float beta[CH], iq[CH], ik[CH];
  const uint32_t D = s.dim, V = s.vdim, tid = threadIdx.x, c0 = blockIdx.x * CH, h = blockIdx.y, P = D + 1u;
  float *qs = lds, *ks = qs + CH * P, *G = ks + CH * P, *vs = G + CH * P;             // G: log2 of the running decay; vs [CH][Vp]
  const uint32_t n_ch = 2u * s.kv_heads * D + s.heads * V, kv = h / (s.heads / s.kv_heads);
  const uint32_t qc = kv * D, kc = s.kv_heads * D + kv * D, vc = 2u * s.kv_heads * D + h * V;
  const float* x = act + s.x;
  const float* ring = state + (uint64_t)seq0 * s.seq_stride + s.conv_off;
  float* out = scratch + ((uint64_t)h * cd.n_chunks + blockIdx.x) * chunk_floats(cd.Dp, cd.Vp);
  float *oW = out, *oQ = oW + CH * cd.Dp, *oK = oQ + CH * cd.Dp, *oB = oK + CH * cd.Dp, *oU = oB + 256u, *oG = oU + CH * cd.Vp;
  for (uint32_t i = tid; i < 2u * D; i += 256u) {
    const bool is_k = i >= D;
    const uint32_t d = is_k ? i - D : i;
    float* to = (is_k ? ks : qs) + d;
    conv_silu_rows<TM>(x, s.x_stride, c0, m, ring, n_ch, (is_k ? kc : qc) + d, pos, act + (is_k ? s.ck : s.cq) + (uint64_t)(kv * D + d) * s.taps,
                       s.taps, [&](int t, float v) { to[t * P] = v; });
  }
  if (tid < CH) beta[tid] = c0 + tid < m ? sigmoid_f(x[(uint64_t)(c0 + tid) * s.x_stride + s.x_b + h]) : 0.f;
  const float ea = expf(act[s.a_log + h]);
  const uint32_t v_items = (V + 63u) & ~63u;                 // whole waves do one or the other
  for (uint32_t i = tid; i < v_items + D; i += 256u) {
    if (i < v_items) {
      if (i < V) conv_silu_rows<TM>(x, s.x_stride, c0, m, ring, n_ch, vc + i, pos, act + s.cv + (uint64_t)(h * V + i) * s.taps, s.taps,
                                    [&](int t, float v) { vs[t * cd.Vp + i] = v; });
    } else {
      const uint32_t d = i - v_items;
      const float bias = act[s.dt_bias + h * D + d];
      float z[CH];
#pragma unroll
      for (int t = 0; t < (int)CH; t++) z[t] = c0 + t < m ? act[dec_out + (uint64_t)(c0 + t) * dec_stride + h * D + d] + bias : 0.f;
      float lg = 0.f;
#pragma unroll
      for (int t = 0; t < (int)CH; t++) {
        if (c0 + t < m) lg -= fminf(ea * softplus_f(z[t]), NO_MEMORY) * 1.44269504f;
        G[t * P + d] = lg;
      }
    }
  }
  __syncthreads();
  {                                                          // lengths of q and k: 8 threads a row, 32 rows
    const uint32_t rr = tid >> 3, sub = tid & 7u;
    const float* v = (rr < CH ? qs : ks) + (rr & (CH - 1u)) * P;
    float ss = 0.f;
    for (uint32_t d = sub; d < D; d += 8u) ss = fmaf(v[d], v[d], ss);
    ss += __shfl_xor(ss, 1, 64); ss += __shfl_xor(ss, 2, 64); ss += __shfl_xor(ss, 4, 64);
    if (sub == 0) (rr < CH ? iq : ik)[rr & (CH - 1u)] = 1.0f / sqrtf(ss + 1e-6f) / (rr < CH ? sqrtf((float)D) : 1.0f);
  }
  __syncthreads();
  {
    const uint32_t t = tid >> 4, r = tid & 15u;
    float a = 0.f, b = 0.f;
    if (r <= t) {
#pragma unroll 4
      for (uint32_t d = 0; d < D; d++) {
        const float e = __builtin_amdgcn_exp2f(G[t * P + d] - G[r * P + d]) * ks[r * P + d];
        a = fmaf(ks[t * P + d], e, a); b = fmaf(qs[t * P + d], e, b);
      }
    }
    A[t][r] = r < t ? a * ik[t] * ik[r] * beta[t] : 0.f;
    oB[t * 16u + r] = b * iq[t] * ik[r];
  }
  __syncthreads();
  if (tid < CH) {                                            // column tid of the inverse, forward substitution
    float y[CH];
#pragma unroll
    for (int t = 0; t < (int)CH; t++) {
      float a = (uint32_t)t == tid ? 1.f : 0.f;
#pragma unroll
      for (int r = 0; r < t; r++) a = fmaf(-A[t][r], y[r], a);
      y[t] = a;
      M[t][tid] = a * beta[tid];
    }
  }
  __syncthreads();
  for (uint32_t i = tid; i < 2u * cd.Dp + cd.Vp; i += 256u) {
    if (i < cd.Dp) {
      const uint32_t d = i;
      const bool in = d < D;
      const float gl = in ? G[15u * P + d] : 0.f;
      float kt[CH];
#pragma unroll
      for (int t = 0; t < (int)CH; t++) {
        const float lg = in ? G[t * P + d] : 0.f;
        oQ[t * cd.Dp + d] = in ? qs[t * P + d] * iq[t] * __builtin_amdgcn_exp2f(lg) : 0.f;
        kt[t] = in ? ks[t * P + d] * ik[t] * __builtin_amdgcn_exp2f(gl - lg) : 0.f;
      }
#pragma unroll
      for (int t = 0; t < (int)CH; t += 4) *(f4_t*)(oK + d * 16u + t) = (f4_t){kt[t], kt[t + 1], kt[t + 2], kt[t + 3]};
      oG[d] = __builtin_amdgcn_exp2f(gl);
    } else {
      const bool is_u = i >= 2u * cd.Dp;
      const uint32_t d = is_u ? i - 2u * cd.Dp : i - cd.Dp;
      float y[CH];
#pragma unroll
      for (int t = 0; t < (int)CH; t++)
        y[t] = is_u ? (d < V ? vs[t * cd.Vp + d] : 0.f) : d < D ? ks[t * P + d] * ik[t] * __builtin_amdgcn_exp2f(G[t * P + d]) : 0.f;
      float* o = is_u ? oU + d : oW + d;
      const uint32_t os = is_u ? cd.Vp : cd.Dp;
#pragma unroll
      for (int t = 0; t < (int)CH; t++) {
        float a = 0.f;
#pragma unroll
        for (int r = 0; r <= t; r++) a = fmaf(M[t][r], y[r], a);
        o[t * os] = a;
      }
    }
  }
}

__global__ void __launch_bounds__(256)
k_retention_prep(const RSpec s, const float* __restrict__ act, float* __restrict__ scratch, ChunkDims cd, uint32_t m, uint32_t pos) {
  extern __shared__ float lds[];
  __shared__ float pw[CH + 1];
  const uint32_t D = s.dim, V = s.vdim, tid = threadIdx.x, c0 = blockIdx.x * CH, h = blockIdx.y, P = D + 1u, half = s.rot_dims >> 1;
  const uint32_t L = min(CH, m - c0);
  float *qs = lds, *ks = qs + CH * P, *cs = ks + CH * P, *sn = cs + CH * half;
  float* out = scratch + ((uint64_t)h * cd.n_chunks + blockIdx.x) * chunk_floats(cd.Dp, cd.Vp);
  float *oQ = out + CH * cd.Dp, *oK = oQ + CH * cd.Dp, *oB = oK + CH * cd.Dp, *oU = oB + 256u, *oG = oU + CH * cd.Vp;
  const float kscale = 1.0f / sqrtf((float)D);
  if (tid == 0) {
    const float dec = act[s.decay + h];
    pw[0] = 1.f;
    for (uint32_t i = 1; i <= CH; i++) pw[i] = pw[i - 1] * dec;
  }
  for (uint32_t i = tid; i < 2u * D; i += 256u) {
    const bool is_k = i >= D;
    const uint32_t d = is_k ? i - D : i;
    const float* src = act + s.x + (is_k ? s.x_k : s.x_q) + h * D + d;
    float* to = (is_k ? ks : qs) + d;
    float v[CH];
#pragma unroll
    for (int t = 0; t < (int)CH; t++) v[t] = c0 + t < m ? src[(uint64_t)(c0 + t) * s.x_stride] : 0.f;
#pragma unroll
    for (int t = 0; t < (int)CH; t++) to[t * P] = is_k ? v[t] * kscale : v[t];
  }
  for (uint32_t i = tid; i < CH * half; i += 256u) {
    const uint32_t t = i / half, d = i - t * half;
    float a, b;
    sincosf((float)(pos + c0 + t) * act[s.freq + d], &a, &b);
    sn[i] = a; cs[i] = b;
  }
  for (uint32_t v = tid; v < cd.Vp; v += 256u) {
    float y[CH];
#pragma unroll
    for (int t = 0; t < (int)CH; t++) y[t] = (c0 + t < m && v < V) ? act[s.x + (uint64_t)(c0 + t) * s.x_stride + s.x_v + h * V + v] : 0.f;
#pragma unroll
    for (int t = 0; t < (int)CH; t++) oU[t * cd.Vp + v] = y[t];
  }
  __syncthreads();
  for (uint32_t i = tid; i < 2u * CH * half; i += 256u) {     // turn the pairs in place
    const bool is_k = i >= CH * half;
    const uint32_t j = is_k ? i - CH * half : i, t = j / half, d = j - t * half;
    float* r = (is_k ? ks : qs) + t * P;
    const float a = r[d], b = r[d + half];
    r[d] = a * cs[j] - b * sn[j];
    r[d + half] = b * cs[j] + a * sn[j];
  }
  __syncthreads();
  {
    const uint32_t t = tid >> 4, r = tid & 15u;
    float b = 0.f;
    if (r <= t) {
#pragma unroll 4
      for (uint32_t d = 0; d < D; d++) b = fmaf(qs[t * P + d], ks[r * P + d], b);
      b *= pw[t - r];
    }
    oB[t * 16u + r] = b;
  }
  for (uint32_t d = tid; d < cd.Dp; d += 256u) {
    float kt[CH];
#pragma unroll
    for (int t = 0; t < (int)CH; t++) {
      oQ[t * cd.Dp + d] = d < D ? qs[t * P + d] * pw[t + 1] : 0.f;
      kt[t] = (d < D && (uint32_t)t < L) ? ks[t * P + d] * pw[L - 1u - min((uint32_t)t, L - 1u)] : 0.f;
    }
#pragma unroll
    for (int t = 0; t < (int)CH; t += 4) *(f4_t*)(oK + d * 16u + t) = (f4_t){kt[t], kt[t + 1], kt[t + 2], kt[t + 3]};
    oG[d] = pw[L];
  }
}

// ---- the walk over the chunks ---------------------------------------------------------------------------------------
// Four waves share the state rows (NT tiles of 16 each); a tile's accumulator holds rows 4 g + i of lane group g, which
// is also how instruction i wants its right operand when the left one is read as four consecutive columns per lane.
struct ScanArgs {
  uint32_t heads, dim, vdim, out, out_stride, s_off, m, pos;
  ChunkDims cd;
  uint32_t kv_heads, taps, conv_off, x, x_stride;     // delta: the convolution's ring is brought up to date here
};
template <int NT> struct ChunkOps { f4_t w[NT], q[NT], k[NT], gl[NT], b; float u[4]; };

template <bool DELTA, int NT>
__device__ __forceinline__ void load_ops(ChunkOps<NT>& o, const float* blk, const ChunkDims& cd, uint32_t wave, uint32_t c, uint32_t kg,
                                         uint32_t v0) {
  const float *pQ = blk + CH * cd.Dp, *pK = pQ + CH * cd.Dp, *pB = pK + CH * cd.Dp, *pU = pB + 256u, *pG = pU + CH * cd.Vp;
#pragma unroll
  for (int j = 0; j < NT; j++) {
    const uint32_t d0 = (wave * NT + j) * 16u;
    if (DELTA) o.w[j] = *(const f4_t*)(blk + c * cd.Dp + d0 + 4u * kg);
    o.q[j] = *(const f4_t*)(pQ + c * cd.Dp + d0 + 4u * kg);
    o.k[j] = *(const f4_t*)(pK + (d0 + c) * 16u + 4u * kg);
    o.gl[j] = *(const f4_t*)(pG + d0 + 4u * kg);
  }
  o.b = *(const f4_t*)(pB + c * 16u + 4u * kg);
#pragma unroll
  for (int i = 0; i < 4; i++) o.u[i] = pU[(4u * kg + i) * cd.Vp + v0 + c];
}

template <bool DELTA, int NT>
__global__ void __launch_bounds__(256)
k_chunk_scan(const ScanArgs a, const float* __restrict__ scratch, float* act, float* state) {
  __shared__ f4_t pb[2][2][4][64];
  const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, c = lane & 15u, kg = lane >> 4;
  const uint32_t h = blockIdx.x, v0 = blockIdx.y * 16u, D = a.dim, V = a.vdim, v = v0 + c;
  const uint32_t bs = chunk_floats(a.cd.Dp, a.cd.Vp);
  const float* blk = scratch + (uint64_t)h * a.cd.n_chunks * bs;
  float* S = state + a.s_off + (uint64_t)h * D * V;
  f4_t st[NT];
#pragma unroll
  for (int j = 0; j < NT; j++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const uint32_t d = (wave * NT + j) * 16u + 4u * kg + i;
      st[j][i] = (a.pos != 0u && d < D && v < V) ? S[(uint64_t)d * V + v] : 0.f;
    }
  ChunkOps<NT> cur, nxt;
  load_ops<DELTA, NT>(cur, blk, a.cd, wave, c, kg, v0);
  for (uint32_t ci = 0; ci < a.cd.n_chunks; ci++) {
    if (ci + 1u < a.cd.n_chunks) load_ops<DELTA, NT>(nxt, blk + (uint64_t)(ci + 1u) * bs, a.cd, wave, c, kg, v0);
    f4_t p1 = {0, 0, 0, 0}, p2 = {0, 0, 0, 0};
#pragma unroll
    for (int j = 0; j < NT; j++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        if (DELTA) p1 = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.w[j][i], st[j][i], p1, 0, 0, 0);
        p2 = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.q[j][i], st[j][i], p2, 0, 0, 0);
      }
    if (DELTA) pb[ci & 1u][0][wave][lane] = p1;
    pb[ci & 1u][1][wave][lane] = p2;
    __syncthreads();
    f4_t u = {cur.u[0], cur.u[1], cur.u[2], cur.u[3]};
    if (DELTA) {
      const f4_t* r = &pb[ci & 1u][0][0][0];
      u -= (r[lane] + r[64 + lane]) + (r[128 + lane] + r[192 + lane]);
    }
    if (wave == 0u) {
      const f4_t* r = &pb[ci & 1u][1][0][0];
      f4_t o = (r[lane] + r[64 + lane]) + (r[128 + lane] + r[192 + lane]);
#pragma unroll
      for (int i = 0; i < 4; i++) o = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.b[i], u[i], o, 0, 0, 0);
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const uint32_t r2 = ci * CH + 4u * kg + i;
        if (r2 < a.m && v < V) act[a.out + (uint64_t)r2 * a.out_stride + h * V + v] = o[i];
      }
    }
#pragma unroll
    for (int j = 0; j < NT; j++) {
      st[j] *= cur.gl[j];
#pragma unroll
      for (int i = 0; i < 4; i++) st[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.k[j][i], u[i], st[j], 0, 0, 0);
    }
    cur = nxt;
  }
#pragma unroll
  for (int j = 0; j < NT; j++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const uint32_t d = (wave * NT + j) * 16u + 4u * kg + i;
      if (d < D && v < V) S[(uint64_t)d * V + v] = st[j][i];
    }
  if (!DELTA) return;
  const uint32_t n_ch = 2u * a.kv_heads * D + a.heads * V, rep = a.heads / a.kv_heads, kv = h / rep;
  for (uint32_t r = a.m > a.taps ? a.m - a.taps : 0u; r < a.m; r++) {
    float* slot = state + a.conv_off + (uint64_t)((a.pos + r) % a.taps) * n_ch;
    const float* x = act + a.x + (uint64_t)r * a.x_stride;
    if (blockIdx.y == 0 && h % rep == 0)
      for (uint32_t d = tid; d < D; d += 256u) {
        slot[kv * D + d] = x[kv * D + d];
        slot[(a.kv_heads + kv) * D + d] = x[(a.kv_heads + kv) * D + d];
      }
    const uint32_t vc = 2u * a.kv_heads * D + h * V + v;
    if (wave == 0u && kg == 0u && v < V) slot[vc] = x[vc];
  }
}

static Scratch g_chunks;
void recurrent_release() { scratch_free(g_chunks); }

static bool rows_ok(uint64_t off, uint64_t stride, uint64_t rows, uint64_t width, uint64_t n_elems) {
  return in_range(off, (rows - 1) * stride + width, n_elems);
}

template <bool DELTA>
static int launch_scan(const ScanArgs& a, float* act, float* state) {
  const dim3 grid(a.heads, cdiv(a.vdim, 16));
  const float* sc = (const float*)g_chunks.p;
  switch (a.cd.Dp / 64u) {
    case 1: k_chunk_scan<DELTA, 1><<<grid, 256, 0, g.stream>>>(a, sc, act, state); break;
    case 2: k_chunk_scan<DELTA, 2><<<grid, 256, 0, g.stream>>>(a, sc, act, state); break;
    case 3: k_chunk_scan<DELTA, 3><<<grid, 256, 0, g.stream>>>(a, sc, act, state); break;
    case 4: k_chunk_scan<DELTA, 4><<<grid, 256, 0, g.stream>>>(a, sc, act, state); break;
    default: return ADAMAH_ERR_INVALID;
  }
  count_launch();
  return check_launch();
}

static LowRank low_rank(const LinSpec& s) { return {s.w, s.k, s.k_stride, s.src, s.src_stride, s.out, s.out_stride}; }

}  // namespace adamah

using namespace adamah;

extern "C" {

int adamah_delta_rule_dev(uint32_t map_act, uint32_t map_opnd, uint32_t map_wt, uint32_t h_spec, uint32_t h_decay, uint32_t h_gate,
                          uint32_t n_seq, uint32_t rows, uint32_t seq0, uint32_t pos) { ADAMAH_API();
  Map *ma = get_f32_map(map_act), *mo = get_map(map_opnd), *mw = get_map(map_wt);
  const DSpec* s = spec_of<DSpec>(h_spec);
  const LinSpec *da = spec_of<LinSpec>(h_decay), *ga = spec_of<LinSpec>(h_gate);
  if (!ma || !mw || mw->dtype != DTYPE_BF16 || !s || !da || !ga || n_seq == 0 || rows == 0 || (n_seq > 1 && rows > 1)) return ADAMAH_ERR_INVALID;
  Map* ms = get_f32_map(s->state_map);
  const uint64_t D = s->dim, V = s->vdim, H = s->heads, KH = s->kv_heads, n_tok = (uint64_t)n_seq * rows;
  if (!ms || D == 0 || D > 256 || V == 0 || H == 0 || KH == 0 || H % KH || s->taps == 0 || s->taps > MAX_TAPS) return ADAMAH_ERR_INVALID;
  const uint64_t n_ch = 2 * KH * D + H * V;
  if (s->x_stride < n_ch || s->x_b + H > s->x_stride) return ADAMAH_ERR_INVALID;
  if (!rows_ok(s->x, s->x_stride, n_tok, s->x_stride, ma->n_elems) || !rows_ok(s->out, s->out_stride, n_tok, H * V, ma->n_elems)) return ADAMAH_ERR_INVALID;
  if (!in_range(s->cq, KH * D * s->taps, ma->n_elems) || !in_range(s->ck, KH * D * s->taps, ma->n_elems) ||
      !in_range(s->cv, H * V * s->taps, ma->n_elems) || !in_range(s->a_log, H, ma->n_elems) || !in_range(s->dt_bias, H * D, ma->n_elems)) return ADAMAH_ERR_INVALID;
  if ((uint64_t)s->s_off + H * D * V > s->seq_stride || (uint64_t)s->conv_off + n_ch * s->taps > s->seq_stride ||
      !in_range((uint64_t)seq0 * s->seq_stride, (uint64_t)n_seq * s->seq_stride, ms->n_elems)) return ADAMAH_ERR_INVALID;
  for (const LinSpec* l : {da, ga}) {
    const uint64_t n = l == da ? H * D : H * V;
    if (l->n != n || l->k == 0 || l->k_stride < l->k || (l->k_stride & 63u) || (l->w & 7u) || l->epi || l->groups ||
        !in_range(l->w, n * l->k_stride, mw->n_elems) || !rows_ok(l->src, l->src_stride, n_tok, l->k, ma->n_elems) ||
        !rows_ok(l->out, l->out_stride, n_tok, n, ma->n_elems)) return ADAMAH_ERR_INVALID;
  }
  float *act = (float*)ma->buf, *state = (float*)ms->buf;
  if (rows == 1) {
    const size_t lds = (size_t)(3 * D + da->k_stride + ga->k_stride) * 4;
    if (lds > 48000) return ADAMAH_ERR_INVALID;
    const dim3 grid((uint32_t)H, cdiv(V, VC), n_seq);
    const bf16_t* W = (const bf16_t*)mw->buf;
#define STEP(DN, TM) k_delta_step<DN, TM><<<grid, DSTEP, lds, g.stream>>>(*s, low_rank(*da), low_rank(*ga), act, W, state, seq0, pos)
    if (s->taps <= 4) { if (D <= 64) STEP(4, 4); else if (D <= 128) STEP(8, 4); else STEP(16, 4); }
    else { if (D <= 64) STEP(4, MAX_TAPS); else if (D <= 128) STEP(8, MAX_TAPS); else STEP(16, MAX_TAPS); }
#undef STEP
    count_launch();
    return check_launch();
  }
  if (int r = adamah_linear_dev(map_act, map_opnd, map_wt, h_decay, 0, rows)) return r;
  if (int r = adamah_linear_dev(map_act, map_opnd, map_wt, h_gate, 0, rows)) return r;
  const ChunkDims cd = {(uint32_t)((D + 63) / 64 * 64), (uint32_t)((V + 15) / 16 * 16), cdiv(rows, CH)};
  if (int r = scratch_need(g_chunks, (size_t)H * cd.n_chunks * chunk_floats(cd.Dp, cd.Vp) * 4)) return r;
  const size_t lds = (size_t)CH * (3 * (D + 1) + cd.Vp) * 4;
  if (lds > 120000) return ADAMAH_ERR_INVALID;
#define PREP(TM)                                                                                                                      \
  do {                                                                                                                                \
    if (lds > 60000) hipFuncSetAttribute((const void*)k_delta_prep<TM>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);         \
    k_delta_prep<TM><<<dim3(cd.n_chunks, (uint32_t)H), 256, lds, g.stream>>>(*s, da->out, da->out_stride, act, state,                 \
                                                                            (float*)g_chunks.p, cd, rows, seq0, pos);                \
  } while (0)
  if (s->taps <= 4) PREP(4); else PREP(MAX_TAPS);
#undef PREP
  count_launch();
  if (int r = check_launch()) return r;
  ScanArgs a = {s->heads, s->dim, s->vdim, s->out, s->out_stride, s->s_off, rows, pos, cd, s->kv_heads, s->taps, s->conv_off, s->x, s->x_stride};
  return launch_scan<true>(a, act, state + (uint64_t)seq0 * s->seq_stride);
}

int adamah_retention_dev(uint32_t map_act, uint32_t h_spec, uint32_t n_seq, uint32_t rows, uint32_t seq0, uint32_t pos) { ADAMAH_API();
  Map* ma = get_f32_map(map_act);
  const RSpec* s = spec_of<RSpec>(h_spec);
  if (!ma || !s || n_seq == 0 || rows == 0 || (n_seq > 1 && rows > 1)) return ADAMAH_ERR_INVALID;
  Map* ms = get_f32_map(s->state_map);
  const uint64_t D = s->dim, V = s->vdim, H = s->heads, n_tok = (uint64_t)n_seq * rows;
  if (!ms || D == 0 || D > 256 || V == 0 || H == 0 || s->rot_dims > D || (s->rot_dims & 1u)) return ADAMAH_ERR_INVALID;
  if (s->x_q + H * D > s->x_stride || s->x_k + H * D > s->x_stride || s->x_v + H * V > s->x_stride ||
      !rows_ok(s->x, s->x_stride, n_tok, s->x_stride, ma->n_elems) || !rows_ok(s->out, s->out_stride, n_tok, H * V, ma->n_elems) ||
      !in_range(s->freq, s->rot_dims / 2, ma->n_elems) || !in_range(s->decay, H, ma->n_elems)) return ADAMAH_ERR_INVALID;
  if ((uint64_t)s->s_off + H * D * V > s->seq_stride ||
      !in_range((uint64_t)seq0 * s->seq_stride, (uint64_t)n_seq * s->seq_stride, ms->n_elems)) return ADAMAH_ERR_INVALID;
  float *act = (float*)ma->buf, *state = (float*)ms->buf;
  if (rows == 1) {
    const dim3 grid((uint32_t)H, cdiv(V, VC), n_seq);
    const size_t lds = (size_t)2 * D * 4;
    if (D <= 64) k_retention_step<8><<<grid, 256, lds, g.stream>>>(*s, act, state, seq0, pos);
    else if (D <= 128) k_retention_step<16><<<grid, 256, lds, g.stream>>>(*s, act, state, seq0, pos);
    else k_retention_step<32><<<grid, 256, lds, g.stream>>>(*s, act, state, seq0, pos);
    count_launch();
    return check_launch();
  }
  const ChunkDims cd = {(uint32_t)((D + 63) / 64 * 64), (uint32_t)((V + 15) / 16 * 16), cdiv(rows, CH)};
  if (int r = scratch_need(g_chunks, (size_t)H * cd.n_chunks * chunk_floats(cd.Dp, cd.Vp) * 4)) return r;
  k_retention_prep<<<dim3(cd.n_chunks, (uint32_t)H), 256, (size_t)CH * (2 * (D + 1) + s->rot_dims) * 4, g.stream>>>(*s, act, (float*)g_chunks.p, cd, rows, pos);
  count_launch();
  if (int r = check_launch()) return r;
  ScanArgs a = {s->heads, s->dim, s->vdim, s->out, s->out_stride, s->s_off, rows, pos, cd, 0, 0, 0, 0, 0};
  return launch_scan<false>(a, act, state + (uint64_t)seq0 * s->seq_stride);
}

}  // extern "C"
