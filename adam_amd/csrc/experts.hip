// Mixture of gated experts over rows whose router logits are known (AdamahExpertsSpec).  Scores, choice and weights are
// float32.
//
// One row: two launches.  Every workgroup chooses the experts for itself (a row of logits is small: each candidate counts
// those that beat it), so nothing has to wait for a launch that only chooses.  k_experts_in: gate and up rows of the chosen
// experts, two matrix rows a wave; k_experts_out: a row of the result is one dot product over the chosen experts'
// activations, already weighted, and the shared expert's behind each other; the row itself times the weights of those that
// give it back is added at the end.
//
// More rows: k_experts_choose (a wave per row), k_experts_list (a workgroup per expert: its rows in order), then the two
// products over tiles of one expert's rows each, k_experts_tiled (bfloat16 operands) or k_experts_f32.  The rows of an
// expert are picked up where they lie; activations and results are laid down so that k_experts_sum can add up a row's in a
// fixed order: what a row gets does not depend on which other rows there are.
#include "linear_common.h"
#include <algorithm>

namespace adamah {

typedef AdamahExpertsSpec XSpec;
#define MAX_CHOICES 1024u
#define MAX_TOP 64u
#define MAX_STEP 32768u      // activations of one row
#define XSTEP 512u

// ---- one row --------------------------------------------------------------------------------------------------------
struct Chosen { float score[MAX_CHOICES], by[MAX_CHOICES]; uint32_t id[MAX_TOP]; float wt[MAX_TOP]; uint32_t n; float back; };
// The chosen experts with matrices, best first, and their weights; n of them; back: what the row itself is multiplied by.
__device__ __forceinline__ void choose_row(const XSpec& s, const float* act, Chosen& ch) {
  const uint32_t tid = threadIdx.x, lane = tid & 63u, n = s.experts + s.identity;
  const float *z = act + s.logits, *corr = act + s.correction;
  float mx = -3.4e38f, sum = 0.f;
  for (uint32_t i = lane; i < n; i += 64u) mx = fmaxf(mx, z[i]);
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
  for (uint32_t i = lane; i < n; i += 64u) sum += expf(z[i] - mx);
  const float inv = 1.0f / wsum64(sum);
  for (uint32_t i = tid; i < n; i += XSTEP) { const float p = expf(z[i] - mx) * inv; ch.score[i] = p; ch.by[i] = p + corr[i]; }
  if (tid < MAX_TOP) { ch.id[tid] = 0xFFFFFFFFu; ch.wt[tid] = 0.f; }
  __syncthreads();
  for (uint32_t i = tid; i < n; i += XSTEP) {
    const float me = ch.by[i];
    uint32_t rank = 0;
#pragma unroll 8
    for (uint32_t j = 0; j < n; j++) rank += ch.by[j] > me || (ch.by[j] == me && j < i) ? 1u : 0u;
    if (rank < s.top) { ch.id[rank] = i; ch.wt[rank] = ch.score[i]; }
  }
  __syncthreads();
  if (tid < 64u) {
    const uint32_t e = ch.id[lane];
    const float w = ch.wt[lane];
    const bool real = e < s.experts;
    const uint64_t mask = __ballot(real);
    const float back = wsum64(real ? 0.f : w);
    const uint32_t at = __popcll(mask & ((1ull << lane) - 1ull));
    if (real) { ch.id[at] = e; ch.wt[at] = w; }              // (one wave: every lane has read its own before)
    if (lane == 0) { ch.n = __popcll(mask); ch.back = back; }
  }
  __syncthreads();
}

__device__ __forceinline__ void fma8(float& a, const uint4& w, const float4& lo, const float4& hi) {
  a = fmaf(bf_lo(w.x), lo.x, a); a = fmaf(bf_hi(w.x), lo.y, a); a = fmaf(bf_lo(w.y), lo.z, a); a = fmaf(bf_hi(w.y), lo.w, a);
  a = fmaf(bf_lo(w.z), hi.x, a); a = fmaf(bf_hi(w.z), hi.y, a); a = fmaf(bf_lo(w.w), hi.z, a); a = fmaf(bf_hi(w.w), hi.w, a);
}

// x in LDS as two planes (elements 0..3 / 4..7 of every eight), so that a lane's two 16-byte reads are conflict free.
#define PLANE(i, half) ((((i) >> 2) & 1u) * (half) + ((i) >> 3) * 4u + ((i) & 3u))

template <int U>
__global__ void __launch_bounds__(XSTEP)
k_experts_in(const bf16_t* __restrict__ W, float* act, const XSpec s) {
  extern __shared__ __attribute__((aligned(16))) float xs[];
  __shared__ Chosen ch;
  const uint32_t lane = threadIdx.x & 63u, wave = threadIdx.x >> 6, kp = s.k_stride, half = kp >> 1, F = (s.ff + 15u) & ~15u;
  for (uint32_t i = threadIdx.x; i < kp; i += XSTEP) xs[PLANE(i, half)] = i < s.width ? act[s.x + i] : 0.f;
  choose_row(s, act, ch);
  const uint32_t n_tasks = ch.n * F;
  for (uint32_t task = blockIdx.x * (XSTEP / 64u) + wave; task < n_tasks; task += gridDim.x * (XSTEP / 64u)) {
    const uint32_t j = task / F, t = task - j * F;
    const bf16_t* wg = W + s.gate_up + (uint64_t)ch.id[j] * s.gate_up_step + (uint64_t)((t >> 4) * 32u + (t & 15u)) * kp;
    const bf16_t* wu = wg + (uint64_t)16u * kp;
    float a = 0.f, b = 0.f;
    for (uint32_t k0 = lane * 8u; k0 < kp; k0 += 512u * U) {
      uint4 p[U], q[U];
#pragma unroll
      for (int u = 0; u < U; u++) {
        const uint32_t k = k0 + 512u * u;
        p[u] = k < kp ? *(const uint4*)(wg + k) : make_uint4(0, 0, 0, 0);
        q[u] = k < kp ? *(const uint4*)(wu + k) : make_uint4(0, 0, 0, 0);
      }
#pragma unroll
      for (int u = 0; u < U; u++) {
        const uint32_t k = k0 + 512u * u;
        if (k >= kp) break;
        const float4 lo = *(const float4*)(xs + (k >> 1)), hi = *(const float4*)(xs + half + (k >> 1));
        fma8(a, p[u], lo, hi); fma8(b, q[u], lo, hi);
      }
    }
    a = wsum64(a); b = wsum64(b);
    if (lane == 0) act[s.act + j * s.ff_stride + t] = silu_f(a) * b;
  }
}

template <int U>
__global__ void __launch_bounds__(XSTEP)
k_experts_out(const bf16_t* __restrict__ W, float* act, const XSpec s, uint32_t magic) {
  extern __shared__ __attribute__((aligned(16))) float xs[];
  __shared__ Chosen ch;
  const uint32_t lane = threadIdx.x & 63u, wave = threadIdx.x >> 6, fs = s.ff_stride;
  choose_row(s, act, ch);
  const uint32_t body = ch.n * fs, kp = body + (s.shared_ff ? s.shared_ff_stride : 0u), half = kp >> 1;
  const float sg = s.shared_ff ? sigmoid_f(act[s.logits + s.experts + s.identity]) : 0.f;
  for (uint32_t i = threadIdx.x; i < kp; i += XSTEP) {
    float v;
    if (i < body) {
      const uint32_t j = __umulhi(i, magic), c = i - j * fs;
      v = c < s.ff ? act[s.act + i] * ch.wt[j] : 0.f;
    } else {
      const uint32_t c = i - body;
      v = c < s.shared_ff ? act[s.shared_act + c] * sg : 0.f;
    }
    xs[PLANE(i, half)] = v;
  }
  __syncthreads();
  const uint32_t n_tasks = (s.width + 1u) >> 1;
  for (uint32_t task = blockIdx.x * (XSTEP / 64u) + wave; task < n_tasks; task += gridDim.x * (XSTEP / 64u)) {
    const uint32_t r0 = task * 2u, r1 = min(r0 + 1u, s.width - 1u);
    float a = 0.f, b = 0.f;
    for (uint32_t k0 = lane * 8u; k0 < kp; k0 += 512u * U) {
      uint4 p[U], q[U];
#pragma unroll
      for (int u = 0; u < U; u++) {
        const uint32_t k = k0 + 512u * u;
        p[u] = q[u] = make_uint4(0, 0, 0, 0);
        if (k < body) {
          const uint32_t j = __umulhi(k, magic), c = k - j * fs;
          const bf16_t* w = W + s.down + (uint64_t)ch.id[j] * s.down_step + c;
          p[u] = *(const uint4*)(w + (uint64_t)r0 * fs); q[u] = *(const uint4*)(w + (uint64_t)r1 * fs);
        } else if (k < kp) {
          const bf16_t* w = W + s.shared_down + (k - body);
          p[u] = *(const uint4*)(w + (uint64_t)r0 * s.shared_ff_stride); q[u] = *(const uint4*)(w + (uint64_t)r1 * s.shared_ff_stride);
        }
      }
#pragma unroll
      for (int u = 0; u < U; u++) {
        const uint32_t k = k0 + 512u * u;
        if (k >= kp) break;
        const float4 lo = *(const float4*)(xs + (k >> 1)), hi = *(const float4*)(xs + half + (k >> 1));
        fma8(a, p[u], lo, hi); fma8(b, q[u], lo, hi);
      }
    }
    a = wsum64(a); b = wsum64(b);
    if (lane < 2u && r0 + lane < s.width) {
      const uint32_t r = r0 + lane;
      const float y = fmaf(ch.back, act[s.x + r], lane ? b : a);
      float* d = act + s.out + r;
      *d = s.epi ? *d + y : y;
    }
  }
}

// ---- more rows ------------------------------------------------------------------------------------------------------
// Entry row * top + j of `ids` / `wts`: the j-th expert of a row, best first, and its weight.
template <int NV>
__global__ void __launch_bounds__(256)
k_experts_choose(const XSpec s, const float* __restrict__ act, uint32_t* __restrict__ ids, float* __restrict__ wts, uint32_t rows) {
  const uint32_t lane = threadIdx.x & 63u, row = blockIdx.x * 4u + (threadIdx.x >> 6), n = s.experts + s.identity;
  if (row >= rows) return;
  const float* z = act + s.logits + (uint64_t)row * s.logits_stride;
  float p[NV], by[NV], mx = -3.4e38f, sum = 0.f;
#pragma unroll
  for (int i = 0; i < NV; i++) { const uint32_t e = lane + 64u * i; p[i] = e < n ? z[e] : -3.4e38f; mx = fmaxf(mx, p[i]); }
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
#pragma unroll
  for (int i = 0; i < NV; i++) { p[i] = lane + 64u * i < n ? expf(p[i] - mx) : 0.f; sum += p[i]; }
  const float inv = 1.0f / wsum64(sum);
#pragma unroll
  for (int i = 0; i < NV; i++) { const uint32_t e = lane + 64u * i; p[i] *= inv; by[i] = e < n ? p[i] + act[s.correction + e] : -3.4e38f; }
  uint32_t gone = 0;                                        // bit i: candidate lane + 64 i has been taken
  for (uint32_t j = 0; j < s.top; j++) {
    float top = -3.4e38f, w = 0.f;
    uint32_t at = 0xFFFFFFFFu;
#pragma unroll
    for (int i = 0; i < NV; i++) {
      const uint32_t e = lane + 64u * i;
      if (e < n && !(gone >> i & 1u) && (at == 0xFFFFFFFFu || by[i] > top)) { top = by[i]; at = e; w = p[i]; }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float t2 = __shfl_xor(top, o, 64), w2 = __shfl_xor(w, o, 64);
      const uint32_t a2 = (uint32_t)__shfl_xor((int)at, o, 64);
      if (a2 != 0xFFFFFFFFu && (at == 0xFFFFFFFFu || t2 > top || (t2 == top && a2 < at))) { top = t2; at = a2; w = w2; }
    }
    if ((at & 63u) == lane) gone |= 1u << (at >> 6);
    if (lane == 0) { ids[(uint64_t)row * s.top + j] = at; wts[(uint64_t)row * s.top + j] = w; }
  }
}

// A workgroup per expert: the entries that chose it, in order, at list + e * rows; cnt[e]: how many.
__global__ void __launch_bounds__(256)
k_experts_list(const uint32_t* __restrict__ ids, uint32_t* __restrict__ list, uint32_t* __restrict__ cnt, uint32_t rows, uint32_t top) {
  __shared__ uint32_t part[4];
  const uint32_t e = blockIdx.x, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, total = rows * top, per = (total + 255u) / 256u;
  const uint32_t lo = min(tid * per, total), hi = min(lo + per, total);
  uint32_t mine = 0;
#pragma unroll 8
  for (uint32_t i = lo; i < hi; i++) mine += ids[i] == e ? 1u : 0u;
  uint32_t at = mine;
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) { const uint32_t u = (uint32_t)__shfl_up((int)at, o, 64); if ((int)lane >= o) at += u; }
  if (lane == 63u) part[wave] = at;
  __syncthreads();
  uint32_t base = 0;
  for (uint32_t w = 0; w < wave; w++) base += part[w];
  if (tid == 255u) cnt[e] = min(base + at, rows);             // (a row takes an expert once)
  at = base + at - mine;
  for (uint32_t i = lo; i < hi; i++)
    if (ids[i] == e && at < rows) list[(uint64_t)e * rows + at++] = i;
}

// Which tile a workgroup has: tiles are numbered expert by expert, within one by matrix rows and then by tokens, so that
// neighbours share the matrix rows; workgroups land on the eight dies in turn, and every die gets a run of neighbours.
// Every wave finds it for itself from the experts' counts.
struct Tile { uint32_t e, count, first, m, n; };     // expert, its rows, its first activation row, tile of tokens / matrix rows
__device__ __forceinline__ bool pick_tile(const uint32_t* __restrict__ cnt, uint32_t experts, uint32_t bm, uint32_t tiles_n, Tile& t) {
  const uint32_t lane = threadIdx.x & 63u;
  uint32_t total = 0;
  for (uint32_t b = 0; b < experts; b += 64u) total += b + lane < experts ? (cnt[b + lane] + bm - 1u) / bm : 0u;
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) total += (uint32_t)__shfl_xor((int)total, o, 64);
  total *= tiles_n;
  const uint32_t per = (total + 7u) / 8u, id = (blockIdx.x & 7u) * per + (blockIdx.x >> 3);
  if ((blockIdx.x >> 3) >= per || id >= total) return false;
  uint32_t tiles = 0, rows = 0;                              // ahead of this run of 64 experts
  for (uint32_t b = 0; b < experts; b += 64u) {
    const uint32_t c = b + lane < experts ? cnt[b + lane] : 0u, mine = (c + bm - 1u) / bm * tiles_n;
    uint32_t ts = mine, rs = c;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const uint32_t u = (uint32_t)__shfl_up((int)ts, o, 64), v = (uint32_t)__shfl_up((int)rs, o, 64);
      if ((int)lane >= o) { ts += u; rs += v; }
    }
    const uint64_t here = __ballot(tiles + ts > id);
    if (here) {
      const int l = __ffsll((unsigned long long)here) - 1;
      const uint32_t tm = (uint32_t)__shfl((int)mine, l, 64) / tiles_n, at = id - (tiles + (uint32_t)__shfl((int)(ts - mine), l, 64));
      t.e = b + (uint32_t)l; t.count = (uint32_t)__shfl((int)c, l, 64); t.first = rows + (uint32_t)__shfl((int)(rs - c), l, 64);
      t.m = at % tm; t.n = at / tm;
      return true;
    }
    tiles += (uint32_t)__shfl((int)ts, 63, 64); rows += (uint32_t)__shfl((int)rs, 63, 64);
  }
  return false;
}
// results: first product -> the operand rows of the activations, second -> a row of `parts` per entry
template <class T>
__device__ __forceinline__ void put_activation(const XSpec& s, T* opnd, uint32_t arow, uint32_t n0, f4_t gt, f4_t up) {
  const uint32_t c = (n0 >> 5) * 16u + (n0 & 15u), F = (s.ff + 15u) & ~15u;
  T* d = opnd + s.act_opnd + (uint64_t)arow * s.ff_stride + c;
#pragma unroll
  for (int i = 0; i < 4; i++) if (c + i < F) d[i] = (T)(silu_f(gt[i]) * up[i]);
}
__device__ __forceinline__ void put_part(const XSpec& s, float* parts, uint32_t entry, uint32_t n0, f4_t v) {
  float* d = parts + (uint64_t)entry * s.width + n0;
#pragma unroll
  for (int i = 0; i < 4; i++) if (n0 + i < s.width) d[i] = v[i];
}

template <int BM, int BN, bool IN>
__global__ void __launch_bounds__(256)
k_experts_tiled(const bf16_t* __restrict__ W, bf16_t* opnd, float* __restrict__ parts, const XSpec s, const uint32_t* __restrict__ list,
                const uint32_t* __restrict__ cnt, uint32_t rows, uint32_t tiles_n) {
  __shared__ __attribute__((aligned(16))) bf16_t la[2 * BN * 64], lb[2 * BM * 64];
  constexpr int NTN = BN / 32, NTM = BM / 32;
  const uint32_t lane = threadIdx.x & 63u, wave = (uint32_t)__builtin_amdgcn_readfirstlane((int)(threadIdx.x >> 6));
  const uint32_t c = lane & 15u, kg = lane >> 4, kp = IN ? s.k_stride : s.ff_stride, n = IN ? 2u * ((s.ff + 15u) & ~15u) : s.width;
  Tile t;
  if (!pick_tile(cnt, s.experts, BM, tiles_n, t)) return;
  const uint32_t m0 = t.m * BM, n0 = t.n * BN, wn = (wave & 1u) * (BN / 2), wm = (wave >> 1) * (BM / 2);
  const bf16_t* We = W + (IN ? s.gate_up + (uint64_t)t.e * s.gate_up_step : s.down + (uint64_t)t.e * s.down_step);
  const uint32_t* le = list + (uint64_t)t.e * rows;
  f4_t acc[NTN][NTM];
  tile_product<BM, BN>(acc, TileRows<BN>(wave, lane, [&](uint32_t r) { return We + (uint64_t)min(n0 + r, n - 1u) * kp; }),
                       TileRows<BM>(wave, lane, [&](uint32_t r) {
                         const uint32_t i = min(m0 + r, t.count - 1u);
                         return opnd + (IN ? s.opnd + (uint64_t)(le[i] / s.top) * kp : s.act_opnd + (uint64_t)(t.first + i) * kp);
                       }), kp, la, lb, wave, lane);
#pragma unroll
  for (int j = 0; j < NTM; j++) {
    const uint32_t i = m0 + wm + 16u * j + c;
    if (i >= t.count) continue;
    if (IN) {
#pragma unroll
      for (int q = 0; q < NTN; q += 2) put_activation(s, opnd, t.first + i, n0 + wn + 16u * q + 4u * kg, acc[q][j], acc[q + 1][j]);
    } else {
      const uint32_t entry = le[i];
#pragma unroll
      for (int q = 0; q < NTN; q++) put_part(s, parts, entry, n0 + wn + 16u * q + 4u * kg, acc[q][j]);
    }
  }
}

template <bool IN>
__global__ void __launch_bounds__(256)
k_experts_f32(const bf16_t* __restrict__ W, float* opnd, float* __restrict__ parts, const XSpec s, const uint32_t* __restrict__ list,
              const uint32_t* __restrict__ cnt, uint32_t rows, uint32_t tiles_n) {
  __shared__ __attribute__((aligned(16))) float la[64][36], lb[64][36];
  const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, c = lane & 15u, kg = lane >> 4;
  const uint32_t kp = IN ? s.k_stride : s.ff_stride, n = IN ? 2u * ((s.ff + 15u) & ~15u) : s.width;
  Tile t;
  if (!pick_tile(cnt, s.experts, 64u, tiles_n, t)) return;
  const uint32_t m0 = t.m * 64u, n0 = t.n * 64u, wn = (wave & 1u) * 32u, wm = (wave >> 1) * 32u, lr = tid >> 2, lc = (tid & 3u) * 8u;
  const bf16_t* We = W + (IN ? s.gate_up + (uint64_t)t.e * s.gate_up_step : s.down + (uint64_t)t.e * s.down_step);
  const uint32_t* le = list + (uint64_t)t.e * rows;
  const uint32_t xi = min(m0 + lr, t.count - 1u);
  f4_t acc[2][2];
  tile_product_f32(acc, We + (uint64_t)min(n0 + lr, n - 1u) * kp + lc,
                   opnd + (IN ? s.opnd + (uint64_t)(le[xi] / s.top) * kp : s.act_opnd + (uint64_t)(t.first + xi) * kp) + lc, kp, la, lb);
#pragma unroll
  for (int j = 0; j < 2; j++) {
    const uint32_t i = m0 + wm + 16u * j + c;
    if (i >= t.count) continue;
    if (IN) put_activation(s, opnd, t.first + i, n0 + wn + 4u * kg, acc[0][j], acc[1][j]);
    else {
      const uint32_t entry = le[i];
#pragma unroll
      for (int q = 0; q < 2; q++) put_part(s, parts, entry, n0 + wn + 16u * q + 4u * kg, acc[q][j]);
    }
  }
}

// A row's results, its own times the weights of the experts that give it back, and the shared expert's.
__global__ void __launch_bounds__(256)
k_experts_sum(const XSpec s, float* act, const float* __restrict__ parts, const uint32_t* __restrict__ ids, const float* __restrict__ wts,
              uint32_t shared, uint32_t shared_stride) {
  __shared__ float w[MAX_TOP];
  __shared__ uint32_t real[MAX_TOP];
  const uint32_t row = blockIdx.x, tid = threadIdx.x;
  if (tid < s.top) { w[tid] = wts[(uint64_t)row * s.top + tid]; real[tid] = ids[(uint64_t)row * s.top + tid] < s.experts ? 1u : 0u; }
  __syncthreads();
  float back = 0.f;
  for (uint32_t j = 0; j < s.top; j++) back += real[j] ? 0.f : w[j];
  const float sg = s.shared_ff ? sigmoid_f(act[s.logits + (uint64_t)row * s.logits_stride + s.experts + s.identity]) : 0.f;
  const float *x = act + s.x + (uint64_t)row * s.x_stride, *sh = act + shared + (uint64_t)row * shared_stride;
  const float* p = parts + (uint64_t)row * s.top * s.width;
  float* d = act + s.out + (uint64_t)row * s.out_stride;
  for (uint32_t i = tid; i < s.width; i += 256u) {
    float y = back * x[i];
#pragma unroll 4
    for (uint32_t j = 0; j < s.top; j++) if (real[j]) y = fmaf(w[j], p[(uint64_t)j * s.width + i], y);
    if (s.shared_ff) y = fmaf(sg, sh[i], y);
    d[i] = s.epi ? d[i] + y : y;
  }
}

static Scratch g_experts;
void experts_release() { scratch_free(g_experts); }

template <bool IN>
static void experts_product(Map* mo, Map* mw, const XSpec& s, float* parts, const uint32_t* list, const uint32_t* cnt, uint32_t rows) {
  const bf16_t* W = (const bf16_t*)mw->buf;
  const uint64_t entries = (uint64_t)rows * s.top;
  const uint32_t n = IN ? 2u * ((s.ff + 15u) & ~15u) : s.width;
  const auto grid = [&](uint32_t bm, uint32_t tiles_n) {       // no more tiles than this, whatever the rows choose
    return cdiv((entries / bm + std::min<uint64_t>(s.experts, entries)) * tiles_n, 8) * 8u;
  };
  if (mo->dtype == DTYPE_F32)
    k_experts_f32<IN><<<grid(64, cdiv(n, 64)), 256, 0, g.stream>>>(W, (float*)mo->buf, parts, s, list, cnt, rows, cdiv(n, 64));
  else if (entries >= (uint64_t)s.experts * 96u)
    k_experts_tiled<128, 128, IN><<<grid(128, cdiv(n, 128)), 256, 0, g.stream>>>(W, (bf16_t*)mo->buf, parts, s, list, cnt, rows, cdiv(n, 128));
  else
    k_experts_tiled<64, 64, IN><<<grid(64, cdiv(n, 64)), 256, 0, g.stream>>>(W, (bf16_t*)mo->buf, parts, s, list, cnt, rows, cdiv(n, 64));
  count_launch();
}

}  // namespace adamah

using namespace adamah;

extern "C" int adamah_experts_dev(uint32_t map_act, uint32_t map_opnd, uint32_t map_wt, uint32_t h_spec, uint32_t h_shared, uint32_t rows) { ADAMAH_API();
  Map *ma = get_f32_map(map_act), *mo = get_map(map_opnd), *mw = get_map(map_wt);
  const XSpec* s = spec_of<XSpec>(h_spec);
  if (!ma || !mw || mw->dtype != DTYPE_BF16 || !s || rows == 0) return ADAMAH_ERR_INVALID;
  const uint64_t E = s->experts, n = E + s->identity, F16 = (s->ff + 15u) / 16u * 16u, fs = s->ff_stride, wd = s->width;
  const uint64_t n_log = n + (s->shared_ff ? 1 : 0), entries = (uint64_t)rows * s->top;
  if (E == 0 || n > MAX_CHOICES || s->top == 0 || s->top > MAX_TOP || s->top > n || s->ff == 0 || fs < F16 || (fs & 63u) || wd == 0) return ADAMAH_ERR_INVALID;
  if (s->k_stride < wd || (s->k_stride & 63u) || s->k_stride > MAX_STEP || ((s->gate_up | s->gate_up_step | s->down | s->down_step) & 7u)) return ADAMAH_ERR_INVALID;
  if (s->gate_up_step < 2 * F16 * s->k_stride || s->down_step < wd * fs || entries > 0x7FFFFFFFull || s->epi > 1u) return ADAMAH_ERR_INVALID;
  const auto rows_ok = [&](uint64_t off, uint64_t stride, uint64_t width) { return in_range(off, (rows - 1) * stride + width, ma->n_elems); };
  if (!in_range(s->gate_up, (E - 1) * s->gate_up_step + 2 * F16 * s->k_stride, mw->n_elems) ||
      !in_range(s->down, (E - 1) * s->down_step + wd * fs, mw->n_elems)) return ADAMAH_ERR_INVALID;
  if (!rows_ok(s->logits, s->logits_stride, n_log) || !in_range(s->correction, n, ma->n_elems) || !rows_ok(s->x, s->x_stride, wd) ||
      !rows_ok(s->out, s->out_stride, wd)) return ADAMAH_ERR_INVALID;
  float* act = (float*)ma->buf;
  const bf16_t* W = (const bf16_t*)mw->buf;
  if (rows == 1) {
    const uint64_t most = std::min<uint64_t>(s->top, E), held = most * fs + (s->shared_ff ? s->shared_ff_stride : 0);
    if (held > MAX_STEP || !in_range(s->act, most * fs, ma->n_elems)) return ADAMAH_ERR_INVALID;
    if (s->shared_ff && (s->shared_ff_stride < s->shared_ff || (s->shared_ff_stride & 63u) || (s->shared_down & 7u) ||
                         !in_range(s->shared_down, wd * s->shared_ff_stride, mw->n_elems) || !in_range(s->shared_act, s->shared_ff, ma->n_elems))) return ADAMAH_ERR_INVALID;
    const uint32_t cu2 = 2u * (uint32_t)g.n_cu, in_grid = std::min<uint32_t>(cdiv(most * F16, XSTEP / 64), cu2), in_lds = s->k_stride * 4u;
    const uint32_t out_grid = std::min<uint32_t>(cdiv(cdiv(wd, 2), XSTEP / 64), cu2), out_lds = (uint32_t)held * 4u;
    const uint32_t magic = (uint32_t)((0x100000000ull + fs - 1) / fs);       // i / fs = umulhi(i, magic) for i <= MAX_STEP
#define LDS_FOR(K, B) if ((B) > 48000) hipFuncSetAttribute((const void*)(K), hipFuncAttributeMaxDynamicSharedMemorySize, (int)(B))
    if (s->k_stride >= 1024u) { LDS_FOR(k_experts_in<4>, in_lds); k_experts_in<4><<<in_grid, XSTEP, in_lds, g.stream>>>(W, act, *s); }
    else k_experts_in<1><<<in_grid, XSTEP, in_lds, g.stream>>>(W, act, *s);
    count_launch();
    if (int r = check_launch()) return r;
    if (held >= 1024u) { LDS_FOR(k_experts_out<4>, out_lds); k_experts_out<4><<<out_grid, XSTEP, out_lds, g.stream>>>(W, act, *s, magic); }
    else k_experts_out<1><<<out_grid, XSTEP, out_lds, g.stream>>>(W, act, *s, magic);
#undef LDS_FOR
    count_launch();
    return check_launch();
  }
  if (!mo || (mo->dtype != DTYPE_BF16 && mo->dtype != DTYPE_F32) || ((s->opnd | s->act_opnd) & 7u)) return ADAMAH_ERR_INVALID;
  if (!in_range(s->opnd, (uint64_t)rows * s->k_stride, mo->n_elems) || !in_range(s->act_opnd, entries * fs, mo->n_elems)) return ADAMAH_ERR_INVALID;
  uint32_t shared = s->x, shared_stride = s->x_stride;
  if (s->shared_ff) {
    const AdamahLinearSpec* sh = spec_of<AdamahLinearSpec>(h_shared);
    if (!sh || sh->n != wd || sh->epi) return ADAMAH_ERR_INVALID;
    if (int r = adamah_linear_dev(map_act, map_opnd, map_wt, h_shared, 0, rows)) return r;      // (checks its own ranges)
    shared = sh->out; shared_stride = sh->out_stride;
  }
  // scratch: results per entry, choices, weights, the experts' lists and counts
  if (int r = scratch_need(g_experts, (entries * wd + 2 * entries + E * rows + E) * 4)) return r;
  float* parts = (float*)g_experts.p;
  uint32_t* ids = (uint32_t*)(parts + entries * wd);
  float* wts = (float*)(ids + entries);
  uint32_t *list = (uint32_t*)(wts + entries), *cnt = list + E * rows;
#define CHOOSE(NV) k_experts_choose<NV><<<cdiv(rows, 4), 256, 0, g.stream>>>(*s, act, ids, wts, rows)
  if (n <= 64) CHOOSE(1); else if (n <= 128) CHOOSE(2); else if (n <= 256) CHOOSE(4); else CHOOSE(16);
#undef CHOOSE
  count_launch();
  if (int r = check_launch()) return r;
  k_experts_list<<<(uint32_t)E, 256, 0, g.stream>>>(ids, list, cnt, rows, s->top);
  count_launch();
  if (int r = check_launch()) return r;
  experts_product<true>(mo, mw, *s, parts, list, cnt, rows);
  if (int r = check_launch()) return r;
  experts_product<false>(mo, mw, *s, parts, list, cnt, rows);
  if (int r = check_launch()) return r;
  k_experts_sum<<<rows, 256, 0, g.stream>>>(*s, act, parts, ids, wts, shared, shared_stride);
  count_launch();
  return check_launch();
}
