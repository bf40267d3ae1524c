// y = W . f(x) over bfloat16 weight maps, f a grouped RMSNorm (with weight and gate; of one row or of the sum of a row and
// a normed one) or nothing.
//
//   one row      k_gemv_bf16: f is computed by every workgroup while it stages x in LDS (float32), weights stream
//                through registers, float32 multiply-adds; store, add to the residual, gate / up pairs combined, or
//                store + best row of the workgroup (arg-max)
//   2..32 rows   k_linear_skinny: bf16 matrix instructions straight from memory, K split over the waves of a workgroup
//   more rows    k_linear_tiled<BM, BN>: bf16 matrix instructions over LDS tiles filled by direct-to-LDS loads
//   float32 operand map: k_linear_f32, the float32 matrix instruction over the widened weights
// Rows of more than one token pass through the operand map (bf16 or float32, rows k_stride apart, zero beyond k):
// k_operand_rows writes f(x) there, unless the producer already did.
#include "linear_common.h"
#include <algorithm>

namespace adamah {

#define LIN_MAX_GROUPS 1024u
#define LIN_MAX_K 32768u
#define NEG_MAX_F (-3.402823466e+38f)

int scratch_need(Scratch& s, size_t bytes) {
  if (bytes <= s.cap) return ADAMAH_OK;
  hipStreamSynchronize(g.stream);
  layout_changed();
  if (s.p) hipFree(s.p);
  s.p = nullptr; s.cap = 0;
  const size_t cap = std::max<size_t>(bytes, (size_t)1 << 20);
  if (hipMalloc((void**)&s.p, cap) != hipSuccess) { (void)hipGetLastError(); return ADAMAH_ERR_MEMORY; }
  s.cap = cap;
  return ADAMAH_OK;
}
void scratch_free(Scratch& s) {
  if (s.p) hipFree(s.p);
  s.p = nullptr; s.cap = 0;
}

// Sum over a workgroup of NW waves; sh: NW floats that no earlier sum still reads.
template <int NW>
__device__ __forceinline__ float block_sum(float v, float* sh) {
  v = wsum64(v);
  if ((threadIdx.x & 63u) == 0) sh[threadIdx.x >> 6] = v;
  __syncthreads();
  v = 0.f;
#pragma unroll
  for (int w = 0; w < NW; w++) v += sh[w];
  return v;
}
// Root mean squares of the row's groups -> inv (with a barrier behind them).
template <int NT, class Val>
__device__ __forceinline__ void group_inverse(const LinSpec& s, float* inv, float* part, Val val) {
  constexpr uint32_t NW = NT / 64;
  const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, gs = s.k / s.groups;
  if (s.groups >= NW) {
    for (uint32_t gi = wave; gi < s.groups; gi += NW) {
      float ss = 0.f;
      for (uint32_t i = lane; i < gs; i += 64u) { const float v = val(gi * gs + i); ss = fmaf(v, v, ss); }
      ss = wsum64(ss);
      if (lane == 0) inv[gi] = 1.0f / sqrtf(ss / (float)gs + s.eps);
    }
    __syncthreads();
  } else {                                    // fewer groups than waves: `sub` waves share a group
    const uint32_t sub = NW / s.groups, gi = wave / sub, sp = wave % sub;
    float ss = 0.f;
    if (gi < s.groups)
      for (uint32_t i = sp * 64u + lane; i < gs; i += sub * 64u) { const float v = val(gi * gs + i); ss = fmaf(v, v, ss); }
    ss = wsum64(ss);
    if (lane == 0) part[wave] = ss;
    __syncthreads();
    if (tid < s.groups) {
      float t = 0.f;
      for (uint32_t j = 0; j < sub; j++) t += part[tid * sub + j];
      inv[tid] = 1.0f / sqrtf(t / (float)gs + s.eps);
    }
    __syncthreads();
  }
}
// f(x) of one row by a workgroup of NT threads; put(i, value) for i in [0, k_stride).  first: this workgroup also stores
// what the spec wants kept.  inv: LDS, LIN_MAX_GROUPS floats, part: LDS, 2 NT / 64 floats.
template <int NT, class Put>
__device__ __forceinline__ void operand_row(const LinSpec& s, float* act, uint32_t row, bool first, float* inv, float* part, Put put) {
  const uint32_t tid = threadIdx.x;
  const float* x = act + s.src + (uint64_t)row * s.src_stride;
  float* keep = act + s.keep + (uint64_t)row * s.keep_stride;
  const bool kept = first && s.kept;
  const float* wt = act + s.wt;
  if (s.branched) {
    // x + the branch's row behind a norm of its own: eight elements a thread stay in registers (a longer row is read again)
    constexpr int R = 8;
    const float *b = act + s.branch + (uint64_t)row * s.branch_stride, *bw = act + s.branch_wt;
    float* res = act + s.res_out + (uint64_t)row * s.res_stride;
    float xv[R], bv[R], wv[R], nv[R], ss = 0.f;
#pragma unroll
    for (int j = 0; j < R; j++) {
      const uint32_t i = tid + (uint32_t)j * NT;
      const bool on = i < s.k;
      bv[j] = on ? b[i] : 0.f; xv[j] = on ? x[i] : 0.f; wv[j] = on ? bw[i] : 0.f; nv[j] = on && s.wt_len ? wt[i] : 0.f;
    }
#pragma unroll
    for (int j = 0; j < R; j++) ss = fmaf(bv[j], bv[j], ss);
    for (uint32_t i = tid + (uint32_t)R * NT; i < s.k; i += NT) ss = fmaf(b[i], b[i], ss);
    const float ib = 1.0f / sqrtf(block_sum<NT / 64>(ss, part) / (float)s.k + s.eps);
    ss = 0.f;
#pragma unroll
    for (int j = 0; j < R; j++) {
      const uint32_t i = tid + (uint32_t)j * NT;
      xv[j] = fmaf(bv[j] * ib, s.wt_add + wv[j], xv[j]);
      if (i < s.k) ss = fmaf(xv[j], xv[j], ss);
    }
    const auto sum_at = [&](uint32_t i) { return fmaf(b[i] * ib, s.wt_add + bw[i], x[i]); };
    for (uint32_t i = tid + (uint32_t)R * NT; i < s.k; i += NT) { const float v = sum_at(i); ss = fmaf(v, v, ss); }
    const float ix = 1.0f / sqrtf(block_sum<NT / 64>(ss, part + NT / 64) / (float)s.k + s.eps);
    const auto done = [&](uint32_t i, float v, float w) {
      if (first && s.branched == 2u) res[i] = v;
      v *= ix;
      if (s.wt_len) v *= s.wt_add + w;
      if (kept) keep[i] = v;
      put(i, v);
    };
#pragma unroll
    for (int j = 0; j < R; j++) {
      const uint32_t i = tid + (uint32_t)j * NT;
      if (i < s.k) done(i, xv[j], nv[j]);
    }
    for (uint32_t i = tid + (uint32_t)R * NT; i < s.k; i += NT) done(i, sum_at(i), s.wt_len ? wt[i] : 0.f);
  } else if (s.groups) {
    const uint32_t gs = s.k / s.groups;
    const float* gt = act + s.gate + (uint64_t)row * s.gate_stride;
    if (s.gate_act == 3u) group_inverse<NT>(s, inv, part, [&](uint32_t i) { return x[i] * silu_f(gt[i]); });
    else group_inverse<NT>(s, inv, part, [&](uint32_t i) { return x[i]; });
    for (uint32_t i = tid; i < s.k; i += NT) {
      float v = x[i];
      if (s.gate_act == 3u) v *= silu_f(gt[i]);
      v *= inv[i / gs];
      if (s.wt_len) v *= s.wt_add + wt[s.wt_len == s.k ? i : i % s.wt_len];
      if (s.gate_act == 1u) v *= sigmoid_f(gt[i]);
      else if (s.gate_act == 2u) v *= silu_f(gt[i]);
      if (kept) keep[i] = v;
      put(i, v);
    }
  } else {
    for (uint32_t i = tid; i < s.k; i += NT) {
      if (kept) keep[i] = x[i];
      put(i, x[i]);
    }
  }
  for (uint32_t i = s.k + tid; i < s.k_stride; i += NT) put(i, 0.f);
}

template <class T>
__global__ void __launch_bounds__(256)
k_operand_rows(const LinSpec s, float* act, T* __restrict__ dst, const uint32_t* __restrict__ row_idx) {
  __shared__ float inv[LIN_MAX_GROUPS];
  __shared__ float part[8];
  T* d = dst + (uint64_t)blockIdx.x * s.k_stride;
  operand_row<256>(s, act, row_idx ? row_idx[blockIdx.x] : blockIdx.x, true, inv, part, [&](uint32_t i, float v) { d[i] = (T)v; });
}

// ---- one row ------------------------------------------------------------------------------------------------------
// A wave takes two matrix rows at a time (for gate / up pairs: row 32 b + j and its partner 16 further on) and walks
// along K, 512 columns a step, U steps in flight.  x in LDS as two planes (elements 0..3 / 4..7 of every eight), so that
// a lane's two 16-byte reads are conflict free.
enum { LEPI_STORE = 0, LEPI_ADD = 1, LEPI_PAIR = 2, LEPI_ARGMAX = 3 };
template <int EPI, int U>
__global__ void __launch_bounds__(512)
k_gemv_bf16(const bf16_t* __restrict__ W, float* act, const LinSpec s, uint32_t n_tasks, const uint32_t* __restrict__ row_idx,
            float* best_val, uint32_t* best_idx) {
  extern __shared__ __attribute__((aligned(16))) float xs[];
  __shared__ float inv[LIN_MAX_GROUPS];
  __shared__ float part[16];
  __shared__ float bv[8];
  __shared__ uint32_t bi[8];
  const uint32_t lane = threadIdx.x & 63u, wave = threadIdx.x >> 6, kp = s.k_stride, half = kp >> 1;
  const uint32_t pairs = EPI == LEPI_PAIR ? (s.n - s.tail) >> 1 : 0u;        // the tail's rows come two a task behind the pairs
  auto rows_of = [&](uint32_t task, uint32_t& r0, uint32_t& r1) {
    if (EPI == LEPI_PAIR && task < pairs) { r0 = (task >> 4) * 32u + (task & 15u); r1 = r0 + 16u; }
    else { r0 = task * 2u; r1 = min(r0 + 1u, s.n - 1u); }     // (2 pairs + 2 (task - pairs) for the tail)
  };
  uint4 p[U], q[U];
  auto fetch = [&](uint32_t r0, uint32_t r1, uint32_t k0) {
#pragma unroll
    for (int u = 0; u < U; u++) {
      const uint32_t k = k0 + 512u * u;
      p[u] = k < kp ? *(const uint4*)(W + (uint64_t)r0 * kp + k) : make_uint4(0, 0, 0, 0);
      q[u] = k < kp ? *(const uint4*)(W + (uint64_t)r1 * kp + k) : make_uint4(0, 0, 0, 0);
    }
  };
  // the first weights are on their way while x is staged, each further step's under the products of the one before
  uint32_t task = blockIdx.x * 8u + wave, k0 = lane * 8u, r0, r1;
  rows_of(min(task, n_tasks - 1u), r0, r1);
  fetch(r0, r1, k0);
  operand_row<512>(s, act, row_idx ? row_idx[0] : 0u, blockIdx.x == 0u, inv, part,
                   [&](uint32_t i, float v) { xs[((i >> 2) & 1u) * half + (i >> 3) * 4u + (i & 3u)] = v; });
  __syncthreads();
  float top = NEG_MAX_F, a0 = 0.f, a1 = 0.f;
  uint32_t top_i = 0xFFFFFFFFu;
  while (task < n_tasks) {
    uint4 cp[U], cq[U];
#pragma unroll
    for (int u = 0; u < U; u++) { cp[u] = p[u]; cq[u] = q[u]; }
    const bool last = k0 - lane * 8u + 512u * U >= kp;              // of this pair of rows
    const uint32_t next = last ? task + gridDim.x * 8u : task, kn = last ? lane * 8u : k0 + 512u * U, c0 = r0;
    if (next < n_tasks) {
      if (last) rows_of(next, r0, r1);
      fetch(r0, r1, kn);
    }
#pragma unroll
    for (int u = 0; u < U; u++) {
      const uint32_t k = k0 + 512u * u;
      if (k >= kp) break;
      const float4 lo = *(const float4*)(xs + (k >> 1)), hi = *(const float4*)(xs + half + (k >> 1));
      a0 = fmaf(bf_lo(cp[u].x), lo.x, a0); a1 = fmaf(bf_lo(cq[u].x), lo.x, a1);
      a0 = fmaf(bf_hi(cp[u].x), lo.y, a0); a1 = fmaf(bf_hi(cq[u].x), lo.y, a1);
      a0 = fmaf(bf_lo(cp[u].y), lo.z, a0); a1 = fmaf(bf_lo(cq[u].y), lo.z, a1);
      a0 = fmaf(bf_hi(cp[u].y), lo.w, a0); a1 = fmaf(bf_hi(cq[u].y), lo.w, a1);
      a0 = fmaf(bf_lo(cp[u].z), hi.x, a0); a1 = fmaf(bf_lo(cq[u].z), hi.x, a1);
      a0 = fmaf(bf_hi(cp[u].z), hi.y, a0); a1 = fmaf(bf_hi(cq[u].z), hi.y, a1);
      a0 = fmaf(bf_lo(cp[u].w), hi.z, a0); a1 = fmaf(bf_lo(cq[u].w), hi.z, a1);
      a0 = fmaf(bf_hi(cp[u].w), hi.w, a0); a1 = fmaf(bf_hi(cq[u].w), hi.w, a1);
    }
    if (last) {
      a0 = wsum64(a0); a1 = wsum64(a1);
      if (EPI == LEPI_PAIR && task < pairs) {
        if (lane == 0) act[s.out + task] = silu_f(a0) * a1;
      } else {
        const uint32_t r = c0 + lane;
        float y = lane ? a1 : a0;
        if (lane < 2u && r < s.n) {
          if (s.biased) y += act[s.bias + r];
          float* d = EPI == LEPI_PAIR ? act + s.tail_out + (r - 2u * pairs) : act + s.out + r;
          *d = EPI == LEPI_ADD ? *d + y : y;
          if (EPI == LEPI_ARGMAX && !isnan(y) && y > top) { top = y; top_i = r; }
        }
      }
      a0 = a1 = 0.f;
    }
    task = next; k0 = kn;
  }
  if (EPI != LEPI_ARGMAX) return;
  const float v1 = __shfl(top, 1, 64);
  const uint32_t i1 = (uint32_t)__shfl((int)top_i, 1, 64);
  if (lane == 0) {
    if (v1 > top || (v1 == top && i1 < top_i)) { top = v1; top_i = i1; }
    bv[wave] = top; bi[wave] = top_i;
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < 8; w++) if (bv[w] > top || (bv[w] == top && bi[w] < top_i)) { top = bv[w]; top_i = bi[w]; }
    best_val[blockIdx.x] = top; best_idx[blockIdx.x] = top_i;
  }
}
// best of n (value, index) pairs; ties to the lower index -> float(index)
__global__ void __launch_bounds__(256)
k_best_pair(const float* __restrict__ val, const uint32_t* __restrict__ idx, uint32_t n, float* dst) {
  __shared__ float sv[4];
  __shared__ uint32_t si[4];
  float v = NEG_MAX_F;
  uint32_t b = 0xFFFFFFFFu;
  for (uint32_t i = threadIdx.x; i < n; i += 256u)
    if (val[i] > v || (val[i] == v && idx[i] < b)) { v = val[i]; b = idx[i]; }
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float tv = __shfl_xor(v, o, 64);
    const uint32_t ti = (uint32_t)__shfl_xor((int)b, o, 64);
    if (tv > v || (tv == v && ti < b)) { v = tv; b = ti; }
  }
  if ((threadIdx.x & 63u) == 0) { sv[threadIdx.x >> 6] = v; si[threadIdx.x >> 6] = b; }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < 4; w++) if (sv[w] > v || (sv[w] == v && si[w] < b)) { v = sv[w]; b = si[w]; }
    *dst = (float)(b == 0xFFFFFFFFu ? 0u : b);
  }
}
// arg-max of every row of a [rows, n] block
__global__ void __launch_bounds__(256)
k_best_row(const float* __restrict__ act, uint64_t src, uint32_t stride, uint32_t n, float* out, const uint32_t* __restrict__ dst) {
  __shared__ float sv[4];
  __shared__ uint32_t si[4];
  const float* x = act + src + (uint64_t)blockIdx.x * stride;
  float v = NEG_MAX_F;
  uint32_t b = 0xFFFFFFFFu;
  for (uint32_t i = threadIdx.x; i < n; i += 256u) { const float t = x[i]; if (t > v) { v = t; b = i; } }
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float tv = __shfl_xor(v, o, 64);
    const uint32_t ti = (uint32_t)__shfl_xor((int)b, o, 64);
    if (tv > v || (tv == v && ti < b)) { v = tv; b = ti; }
  }
  if ((threadIdx.x & 63u) == 0) { sv[threadIdx.x >> 6] = v; si[threadIdx.x >> 6] = b; }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < 4; w++) if (sv[w] > v || (sv[w] == v && si[w] < b)) { v = sv[w]; b = si[w]; }
    out[dst[blockIdx.x]] = (float)(b == 0xFFFFFFFFu ? 0u : b);
  }
}

// ---- results of the matrix-instruction kernels --------------------------------------------------------------------
// Lane l of a 16 x 16 result holds matrix rows (outputs) 4 (l / 16) + 0..3 of token l % 16.
__device__ __forceinline__ void put_out(const LinSpec& s, float* act, uint32_t row, uint32_t n0, f4_t v) {
  float* d = act + s.out + (uint64_t)row * s.out_stride + n0;
  if (s.biased) {
#pragma unroll
    for (int i = 0; i < 4; i++) if (n0 + i < s.n) v[i] += act[s.bias + n0 + i];
  }
  if (s.epi == 1u) {
#pragma unroll
    for (int i = 0; i < 4; i++) if (n0 + i < s.n) d[i] += v[i];
  } else {
#pragma unroll
    for (int i = 0; i < 4; i++) if (n0 + i < s.n) d[i] = v[i];
  }
}
// gate rows n0 .. n0 + 3 and their up rows -> the activation's operand rows
template <class T>
__device__ __forceinline__ void put_pair(const LinSpec& s, T* opnd, uint32_t row, uint32_t n0, f4_t gt, f4_t up) {
  const uint32_t c = (n0 >> 5) * 16u + (n0 & 15u);
  T* d = opnd + s.out_opnd + (uint64_t)row * s.out_opnd_stride + c;
#pragma unroll
  for (int i = 0; i < 4; i++) if (n0 + i < s.n) d[i] = (T)(silu_f(gt[i]) * up[i]);
}
// two neighbouring runs of 16 rows of an epi 2 product, from row n0 on: a pair, or two runs of the tail
template <class T>
__device__ __forceinline__ void put_pair_or_tail(const LinSpec& s, float* act, T* opnd, uint32_t row, uint32_t n0, f4_t a, f4_t b) {
  const uint32_t head = s.n - s.tail;
  if (n0 < head) { put_pair(s, opnd, row, n0, a, b); return; }
  float* d = act + s.tail_out + (uint64_t)row * s.tail_stride + (n0 - head);
#pragma unroll
  for (int i = 0; i < 4; i++) {
    if (n0 + i < s.n) d[i] = a[i];
    if (n0 + 16u + i < s.n) d[16 + i] = b[i];
  }
}

// ---- 2 .. 32 rows -------------------------------------------------------------------------------------------------
// A workgroup owns 32 matrix rows; its 8 waves take 32-column steps of K in turn and add up through LDS.
template <int MT>
__global__ void __launch_bounds__(512)
k_linear_skinny(const bf16_t* __restrict__ W, const bf16_t* __restrict__ X, float* act, bf16_t* opnd, const LinSpec s, uint32_t rows) {
  __shared__ f4_t red[8][2 * MT][64];
  const uint32_t lane = threadIdx.x & 63u, wave = threadIdx.x >> 6, c = lane & 15u, kg = lane >> 4, kp = s.k_stride;
  const uint32_t n0 = blockIdx.x * 32u;
  const bf16_t* wa = W + (uint64_t)min(n0 + c, s.n - 1u) * kp + kg * 8u;
  const bf16_t* wb = W + (uint64_t)min(n0 + 16u + c, s.n - 1u) * kp + kg * 8u;
  const bf16_t* xr[MT];
#pragma unroll
  for (int m = 0; m < MT; m++) xr[m] = X + (uint64_t)min(16u * m + c, rows - 1u) * kp + kg * 8u;
  f4_t acc[2][MT];
#pragma unroll
  for (int m = 0; m < MT; m++) { acc[0][m] = (f4_t){0, 0, 0, 0}; acc[1][m] = (f4_t){0, 0, 0, 0}; }
  constexpr int UN = 4;                                // K steps in flight
  for (uint32_t k0 = wave * 32u; k0 < kp; k0 += 256u * UN) {
    bf8_t a[UN], b[UN], x[UN][MT];
#pragma unroll
    for (int u = 0; u < UN; u++) {
      const uint32_t k = min(k0 + 256u * u, kp - 32u);
      a[u] = *(const bf8_t*)(wa + k); b[u] = *(const bf8_t*)(wb + k);
#pragma unroll
      for (int m = 0; m < MT; m++) x[u][m] = *(const bf8_t*)(xr[m] + k);
    }
#pragma unroll
    for (int u = 0; u < UN; u++) {
      if (k0 + 256u * u >= kp) break;
#pragma unroll
      for (int m = 0; m < MT; m++) {
        acc[0][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[u], x[u][m], acc[0][m], 0, 0, 0);
        acc[1][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(b[u], x[u][m], acc[1][m], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int m = 0; m < MT; m++) { red[wave][m][lane] = acc[0][m]; red[wave][MT + m][lane] = acc[1][m]; }
  __syncthreads();
  if (s.epi == 2u) {
    if (wave < MT) {
      f4_t gt = red[0][wave][lane], up = red[0][MT + wave][lane];
      for (int w = 1; w < 8; w++) { gt += red[w][wave][lane]; up += red[w][MT + wave][lane]; }
      const uint32_t row = 16u * wave + c;
      if (row < rows) put_pair_or_tail(s, act, opnd, row, n0 + 4u * kg, gt, up);
    }
  } else if (wave < 2 * MT) {
    f4_t v = red[0][wave][lane];
    for (int w = 1; w < 8; w++) v += red[w][wave][lane];
    const uint32_t row = 16u * (wave % MT) + c;
    if (row < rows) put_out(s, act, row, n0 + 16u * (wave / MT) + 4u * kg, v);
  }
}

// ---- tiles --------------------------------------------------------------------------------------------------------
template <int BM, int BN>
__global__ void __launch_bounds__(256)
k_linear_tiled(const bf16_t* __restrict__ W, const bf16_t* __restrict__ X, float* act, bf16_t* opnd, const LinSpec s, uint32_t rows,
               uint32_t tiles_m, uint32_t tiles_n) {
  __shared__ __attribute__((aligned(16))) bf16_t la[2 * BN * 64], lb[2 * BM * 64];
  constexpr int NTN = BN / 32, NTM = BM / 32;
  const uint32_t lane = threadIdx.x & 63u, wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6));
  const uint32_t c = lane & 15u, kg = lane >> 4, kp = s.k_stride;
  // workgroups land on the eight dies in turn: give every die a run of neighbouring tiles
  const uint32_t total = tiles_m * tiles_n, per = (total + 7u) / 8u;
  const uint32_t id = (blockIdx.x & 7u) * per + (blockIdx.x >> 3);
  if (id >= total || (blockIdx.x >> 3) >= per) return;
  const uint32_t m0 = (id % tiles_m) * BM, n0 = (id / tiles_m) * BN;
  const uint32_t wn = (wave & 1u) * (BN / 2), wm = (wave >> 1) * (BM / 2);
  f4_t acc[NTN][NTM];
  tile_product<BM, BN>(acc, TileRows<BN>(wave, lane, [&](uint32_t r) { return W + (uint64_t)min(n0 + r, s.n - 1u) * kp; }),
                       TileRows<BM>(wave, lane, [&](uint32_t r) { return X + (uint64_t)min(m0 + r, rows - 1u) * kp; }), kp, la, lb, wave, lane);
#pragma unroll
  for (int j = 0; j < NTM; j++) {
    const uint32_t row = m0 + wm + 16u * j + c;
    if (row >= rows) continue;
    if (s.epi == 2u) {
#pragma unroll
      for (int i = 0; i < NTN; i += 2) put_pair_or_tail(s, act, opnd, row, n0 + wn + 16u * i + 4u * kg, acc[i][j], acc[i + 1][j]);
    } else {
#pragma unroll
      for (int i = 0; i < NTN; i++) put_out(s, act, row, n0 + wn + 16u * i + 4u * kg, acc[i][j]);
    }
  }
}

// ---- float32 operands ---------------------------------------------------------------------------------------------
__global__ void __launch_bounds__(256)
k_linear_f32(const bf16_t* __restrict__ W, const float* __restrict__ X, float* act, float* opnd, const LinSpec s, uint32_t rows) {
  __shared__ __attribute__((aligned(16))) float la[64][36], lb[64][36];
  const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, c = lane & 15u, kg = lane >> 4, kp = s.k_stride;
  const uint32_t m0 = blockIdx.y * 64u, n0 = blockIdx.x * 64u, wn = (wave & 1u) * 32u, wm = (wave >> 1) * 32u;
  const uint32_t lr = tid >> 2, lc = (tid & 3u) * 8u;
  const bf16_t* wsrc = W + (uint64_t)min(n0 + lr, s.n - 1u) * kp + lc;
  const float* xsrc = X + (uint64_t)min(m0 + lr, rows - 1u) * kp + lc;
  f4_t acc[2][2];
  tile_product_f32(acc, wsrc, xsrc, kp, la, lb);
#pragma unroll
  for (int j = 0; j < 2; j++) {
    const uint32_t row = m0 + wm + 16u * j + c;
    if (row >= rows) continue;
    if (s.epi == 2u) put_pair_or_tail(s, act, opnd, row, n0 + wn + 4u * kg, acc[0][j], acc[1][j]);
    else
#pragma unroll
      for (int i = 0; i < 2; i++) put_out(s, act, row, n0 + wn + 16u * i + 4u * kg, acc[i][j]);
  }
}

// ---- launch -------------------------------------------------------------------------------------------------------
static Scratch g_best;
void linear_release() { scratch_free(g_best); }

static bool span_ok(uint64_t off, uint64_t stride, uint64_t rows, uint64_t width, uint64_t n_elems) {
  return rows == 0 || in_range(off, (rows - 1) * stride + width, n_elems);
}

static int check_linear(Map* ma, Map* mo, Map* mw, const LinSpec& s, uint32_t rows, uint32_t src_rows) {
  if (!ma || !mw || mw->dtype != DTYPE_BF16 || rows == 0 || s.k == 0 || s.n == 0) return ADAMAH_ERR_INVALID;
  if (s.k_stride < s.k || (s.k_stride & 63u) || (s.w & 7u) || s.k_stride > LIN_MAX_K || s.epi > 2u) return ADAMAH_ERR_INVALID;
  if (!span_ok(s.w, s.k_stride, s.n, s.k_stride, mw->n_elems)) return ADAMAH_ERR_INVALID;
  if (s.groups > LIN_MAX_GROUPS || (s.groups && s.k % s.groups) || (s.gate_act && !s.groups) || (s.wt_len && !s.groups)) return ADAMAH_ERR_INVALID;
  if (!(rows > 1 && s.ready) && !span_ok(s.src, s.src_stride, src_rows, s.k, ma->n_elems)) return ADAMAH_ERR_INVALID;
  if (s.wt_len && !in_range(s.wt, s.wt_len, ma->n_elems)) return ADAMAH_ERR_INVALID;
  if (s.gate_act && !span_ok(s.gate, s.gate_stride, src_rows, s.k, ma->n_elems)) return ADAMAH_ERR_INVALID;
  if (s.tail > s.n || (s.tail && s.epi != 2u) || (s.epi == 2u && ((s.n - s.tail) & 31u)) || s.gate_act > 3u) return ADAMAH_ERR_INVALID;
  if (s.tail && !span_ok(s.tail_out, s.tail_stride, rows, s.tail, ma->n_elems)) return ADAMAH_ERR_INVALID;
  if (s.biased && (s.epi == 2u || !in_range(s.bias, s.n, ma->n_elems))) return ADAMAH_ERR_INVALID;
  if (!(rows > 1 && s.ready)) {
    if (s.branched > 2u || (s.branched && (s.groups != 1u || s.gate_act || (s.wt_len && s.wt_len != s.k)))) return ADAMAH_ERR_INVALID;
    if (s.branched && (!span_ok(s.branch, s.branch_stride, src_rows, s.k, ma->n_elems) || !in_range(s.branch_wt, s.k, ma->n_elems))) return ADAMAH_ERR_INVALID;
    if (s.branched == 2u) {                 // workgroups read src while one of them writes the sum
      if (!span_ok(s.res_out, s.res_stride, src_rows, s.k, ma->n_elems)) return ADAMAH_ERR_INVALID;
      for (const auto& r : {std::make_pair(s.src, s.src_stride), std::make_pair(s.branch, s.branch_stride)}) {
        const uint64_t e0 = s.res_out + (uint64_t)(src_rows - 1) * s.res_stride + s.k, e1 = r.first + (uint64_t)(src_rows - 1) * r.second + s.k;
        if (s.res_out < e1 && r.first < e0) return ADAMAH_ERR_INVALID;
      }
    }
    if (s.kept && !span_ok(s.keep, s.keep_stride, src_rows, s.k, ma->n_elems)) return ADAMAH_ERR_INVALID;
  }
  if (rows > 1) {
    if (!mo || (mo->dtype != DTYPE_BF16 && mo->dtype != DTYPE_F32) || (s.opnd & 7u)) return ADAMAH_ERR_INVALID;
    if (!span_ok(s.opnd, s.k_stride, rows, s.k_stride, mo->n_elems)) return ADAMAH_ERR_INVALID;
  }
  if (s.epi == 2u && rows > 1) return span_ok(s.out_opnd, s.out_opnd_stride, rows, (s.n - s.tail) / 2, mo->n_elems) ? ADAMAH_OK : ADAMAH_ERR_INVALID;
  return span_ok(s.out, s.out_stride, rows, s.epi == 2u ? (s.n - s.tail) / 2 : s.n, ma->n_elems) ? ADAMAH_OK : ADAMAH_ERR_INVALID;
}

static uint32_t gemv_grid(uint32_t n_tasks) { return std::min<uint32_t>(cdiv(n_tasks, 8), 2u * (uint32_t)g.n_cu); }

template <int EPI>
static void gemv_launch(Map* ma, Map* mw, const LinSpec& s, const uint32_t* row_idx, uint32_t n_tasks) {
  const uint32_t grid = gemv_grid(n_tasks);
  const size_t lds = (size_t)s.k_stride * 4;
  const bf16_t* W = (const bf16_t*)mw->buf + s.w;
  float* bv = (float*)g_best.p;
  uint32_t* bi = bv ? (uint32_t*)(bv + grid) : nullptr;
  if (s.k_stride >= 1024u) {
    if (lds > 60000) hipFuncSetAttribute((const void*)k_gemv_bf16<EPI, 4>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    k_gemv_bf16<EPI, 4><<<grid, 512, lds, g.stream>>>(W, (float*)ma->buf, s, n_tasks, row_idx, bv, bi);
  } else k_gemv_bf16<EPI, 1><<<grid, 512, lds, g.stream>>>(W, (float*)ma->buf, s, n_tasks, row_idx, bv, bi);
  count_launch();
}

int run_linear(Map* ma, Map* mo, Map* mw, const LinSpec& s, const uint32_t* row_idx, uint32_t rows) {
  float* act = (float*)ma->buf;
  if (rows == 1) {
    if (s.epi == 2u) gemv_launch<LEPI_PAIR>(ma, mw, s, row_idx, (s.n - s.tail) / 2 + cdiv(s.tail, 2));
    else if (s.epi == 1u) gemv_launch<LEPI_ADD>(ma, mw, s, row_idx, cdiv(s.n, 2));
    else gemv_launch<LEPI_STORE>(ma, mw, s, row_idx, cdiv(s.n, 2));
    return check_launch();
  }
  const bf16_t* W = (const bf16_t*)mw->buf + s.w;
  if (mo->dtype == DTYPE_F32) {
    float* op = (float*)mo->buf;
    if (!s.ready) { k_operand_rows<float><<<rows, 256, 0, g.stream>>>(s, act, op + s.opnd, row_idx); count_launch(); }
    k_linear_f32<<<dim3(cdiv(s.n, 64), cdiv(rows, 64)), 256, 0, g.stream>>>(W, op + s.opnd, act, op, s, rows);
    count_launch();
    return check_launch();
  }
  bf16_t* op = (bf16_t*)mo->buf;
  const bf16_t* X = op + s.opnd;
  if (!s.ready) { k_operand_rows<bf16_t><<<rows, 256, 0, g.stream>>>(s, act, op + s.opnd, row_idx); count_launch(); }
  if (rows <= 16) k_linear_skinny<1><<<cdiv(s.n, 32), 512, 0, g.stream>>>(W, X, act, op, s, rows);
  else if (rows <= 32) k_linear_skinny<2><<<cdiv(s.n, 32), 512, 0, g.stream>>>(W, X, act, op, s, rows);
  else {
    const uint32_t big = cdiv(rows, 128) * cdiv(s.n, 128);
    if (big >= (uint32_t)g.n_cu * 3 / 4) {
      k_linear_tiled<128, 128><<<cdiv(big, 8) * 8, 256, 0, g.stream>>>(W, X, act, op, s, rows, cdiv(rows, 128), cdiv(s.n, 128));
    } else {
      const uint32_t small = cdiv(rows, 64) * cdiv(s.n, 64);
      k_linear_tiled<64, 64><<<cdiv(small, 8) * 8, 256, 0, g.stream>>>(W, X, act, op, s, rows, cdiv(rows, 64), cdiv(s.n, 64));
    }
  }
  count_launch();
  return check_launch();
}

// Rows of a linear op named by a handle: every index must be known on the host, so that the largest can be checked.
static int row_list(uint32_t h_rows, uint32_t rows, const uint32_t** dev, uint32_t* src_rows) {
  *dev = nullptr; *src_rows = rows;
  if (!h_rows) return ADAMAH_OK;
  const uint32_t* hp = res_host(h_rows, rows);
  *dev = res_u32(h_rows, rows);
  if (!hp || !*dev) return ADAMAH_ERR_INVALID;
  *src_rows = *std::max_element(hp, hp + rows) + 1u;
  return ADAMAH_OK;
}

// k_merge_norm: dst += scale * sum over the two parts of rms(part) * weight
template <int NT>
__global__ void __launch_bounds__(NT)
k_merge_norm(const AdamahMergeSpec s, float* act) {
  __shared__ float sh[2][NT / 64];
  const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
  const float* a = act + s.a + (uint64_t)blockIdx.x * s.stride;
  const float* b = act + s.b + (uint64_t)blockIdx.x * s.stride;
  float* d = act + s.dst + (uint64_t)blockIdx.x * s.dst_stride;
  float sa = 0.f, sb = 0.f;
#pragma unroll 4
  for (uint32_t i = tid; i < s.dim; i += NT) { sa = fmaf(a[i], a[i], sa); sb = fmaf(b[i], b[i], sb); }
  sa = wsum64(sa); sb = wsum64(sb);
  if (lane == 0) { sh[0][wave] = sa; sh[1][wave] = sb; }
  __syncthreads();
  sa = sb = 0.f;
#pragma unroll
  for (int w = 0; w < NT / 64; w++) { sa += sh[0][w]; sb += sh[1][w]; }
  const float ia = 1.0f / sqrtf(sa / (float)s.dim + s.eps), ib = 1.0f / sqrtf(sb / (float)s.dim + s.eps);
#pragma unroll 4
  for (uint32_t i = tid; i < s.dim; i += NT) d[i] = (s.store ? 0.f : d[i]) + s.scale * (a[i] * ia * act[s.wa + i] + b[i] * ib * act[s.wb + i]);
}

}  // namespace adamah

using namespace adamah;

extern "C" {

int adamah_linear_dev(uint32_t map_act, uint32_t map_opnd, uint32_t map_wt, uint32_t h_spec, uint32_t h_rows, uint32_t rows) { ADAMAH_API();
  Map *ma = get_f32_map(map_act), *mo = get_map(map_opnd), *mw = get_map(map_wt);
  const LinSpec* s = spec_of<LinSpec>(h_spec);
  const uint32_t* dev;
  uint32_t src_rows;
  if (!s) return ADAMAH_ERR_INVALID;
  if (int r = row_list(h_rows, rows, &dev, &src_rows)) return r;
  if (int r = check_linear(ma, mo, mw, *s, rows, src_rows)) return r;
  return run_linear(ma, mo, mw, *s, dev, rows);
}

int adamah_linear_argmax_dev(uint32_t map_act, uint32_t map_opnd, uint32_t map_wt, uint32_t h_spec, uint32_t h_dst, uint32_t rows) { ADAMAH_API();
  Map *ma = get_f32_map(map_act), *mo = get_map(map_opnd), *mw = get_map(map_wt);
  const LinSpec* s = spec_of<LinSpec>(h_spec);
  if (!s || s->epi != 0u) return ADAMAH_ERR_INVALID;
  if (int r = check_linear(ma, mo, mw, *s, rows, rows)) return r;
  const uint32_t* dst = res_host(h_dst, rows);
  if (!dst) return ADAMAH_ERR_INVALID;
  for (uint32_t i = 0; i < rows; i++) if (dst[i] >= ma->n_elems) return ADAMAH_ERR_INVALID;
  float* act = (float*)ma->buf;
  if (rows == 1) {
    const uint32_t n_tasks = cdiv(s->n, 2), grid = gemv_grid(n_tasks);
    if (int r = scratch_need(g_best, (size_t)grid * 8)) return r;
    gemv_launch<LEPI_ARGMAX>(ma, mw, *s, nullptr, n_tasks);
    k_best_pair<<<1, 256, 0, g.stream>>>((const float*)g_best.p, (const uint32_t*)g_best.p + grid, grid, act + dst[0]);
  } else {
    if (int r = run_linear(ma, mo, mw, *s, nullptr, rows)) return r;
    k_best_row<<<rows, 256, 0, g.stream>>>(act, s->out, s->out_stride, s->n, act, res_u32(h_dst, rows));
  }
  count_launch();
  return check_launch();
}

int adamah_merge_norm_dev(uint32_t map_act, uint32_t h_spec, uint32_t rows) { ADAMAH_API();
  Map* ma = get_f32_map(map_act);
  const AdamahMergeSpec* s = spec_of<AdamahMergeSpec>(h_spec);
  if (!ma || !s || rows == 0 || s->dim == 0) return ADAMAH_ERR_INVALID;
  if (!span_ok(s->a, s->stride, rows, s->dim, ma->n_elems) || !span_ok(s->b, s->stride, rows, s->dim, ma->n_elems) ||
      !span_ok(s->dst, s->dst_stride, rows, s->dim, ma->n_elems) || !in_range(s->wa, s->dim, ma->n_elems) ||
      !in_range(s->wb, s->dim, ma->n_elems)) return ADAMAH_ERR_INVALID;
  if (rows < 64) k_merge_norm<1024><<<rows, 1024, 0, g.stream>>>(*s, (float*)ma->buf);
  else k_merge_norm<256><<<rows, 256, 0, g.stream>>>(*s, (float*)ma->buf);
  count_launch();
  return check_launch();
}

}  // extern "C"
