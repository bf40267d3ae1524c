// State-space recurrence (Mamba-2): one decay per head and token, inputs, B and C behind a short convolution, B and C shared
// by the heads of a group.  S_t = a_t S_(t-1) + dt_t B_t x_t^T, y_t = S_t^T C_t + D x_t, a_t = exp(-exp(A_log) dt_t); state,
// step sizes, decays and every product with the state are float32.
//
// One token (decode): k_space_step.  A workgroup owns one head and 32 of its value columns, which are independent but for
// the convolved B and C that every workgroup of a group makes for itself, so no workgroup waits for another.
//
// A portion of a prompt: two launches.  k_space_prep, a workgroup per chunk of 16 tokens and group or head, writes what the
// chunks are made of: per group C [16, N], B^T [N, 16] and the products C_t . B_s; per head the convolved inputs and, with
// L_t the sum of the decays' logarithms up to token t of the chunk, exp(L_t - L_s) dt_s for s <= t, exp(L_t) and
// exp(L_last - L_s) dt_s.  k_space_scan, a workgroup per head and 16 value columns, walks over the chunks with the state in
// the accumulators of the float32 matrix instruction:
//   y_t = exp(L_t) S^T C_t + sum_{s <= t} (C_t . B_s) exp(L_t - L_s) dt_s x_s + D x_t
//   S  <- exp(L_last) S + sum_s B_s (exp(L_last - L_s) dt_s x_s)^T
// A decay is one number per head and token, so it multiplies results and the 16 input rows; the wide operands stay those of
// the group.  Every exponent is <= 0: no strength of decay overflows.
#include "recurrent_common.h"
#include <algorithm>

namespace adamah {

typedef AdamahStateSpaceSpec SSpec;
#define SSTEP 512u

// One token of one sequence per blockIdx.z; DN: state rows a thread holds (N <= 16 DN); TM >= taps.
template <int DN, int TM>
__global__ void __launch_bounds__(SSTEP)
k_space_step(const SSpec s, float* act, float* state, uint32_t seq0, uint32_t pos) {
  constexpr uint32_t NG = SSTEP / VC;
  __shared__ float bc[2][16 * DN], red[NG][VC], xs[VC];
  const uint32_t N = s.state, V = s.vdim, tid = threadIdx.x, h = blockIdx.x, v0 = blockIdx.y * VC, row = blockIdx.z;
  const uint32_t inner = s.heads * V, n_ch = inner + 2u * s.groups * N, rep = s.heads / s.groups, grp = h / rep;
  const float* xr = act + s.x + (uint64_t)row * s.x_stride;
  const float* x = xr + s.x_c;
  float* ring = state + (uint64_t)(seq0 + row) * s.seq_stride + s.conv_off;
  float* S = state + (uint64_t)(seq0 + row) * s.seq_stride + s.s_off + (uint64_t)h * N * V;
  const uint32_t bch = inner + grp * N, cch = inner + (s.groups + grp) * N, xch = h * V + v0;
  const uint32_t col = tid & (VC - 1u), dg = tid / VC, v = v0 + col;
  float st[DN];
#pragma unroll
  for (int i = 0; i < DN; i++) {
    const uint32_t d = dg + NG * i;
    st[i] = (pos != 0u && d < N && v < V) ? S[(uint64_t)d * V + v] : 0.f;
  }
  const float z = xr[s.x_dt + h] + act[s.dt_bias + h], a_log = act[s.a_log + h], skip = act[s.skip + h];
  for (uint32_t i = tid; i < 2u * N; i += SSTEP) {
    const bool is_c = i >= N;
    const uint32_t d = is_c ? i - N : i, ch = (is_c ? cch : bch) + d;
    bc[is_c ? 1 : 0][d] = conv_silu_ring<TM>(x, ring, n_ch, ch, pos, act + s.conv + (uint64_t)ch * s.taps, s.taps, act[s.conv_b + ch]);
  }
  const uint32_t last = SSTEP - 1u - tid;                     // the inputs: by the threads at the other end
  if (last < VC && v0 + last < V) {
    const uint32_t ch = xch + last;
    xs[last] = conv_silu_ring<TM>(x, ring, n_ch, ch, pos, act + s.conv + (uint64_t)ch * s.taps, s.taps, act[s.conv_b + ch]);
  }
  const float dt = softplus_f(z), keep = expf(-fminf(expf(a_log) * dt, NO_MEMORY));
  __syncthreads();
  const float xv = v < V ? xs[col] : 0.f, dx = dt * xv;
  float y = 0.f;
#pragma unroll
  for (int i = 0; i < DN; i++) {
    const uint32_t d = dg + NG * i;
    if (d < N && v < V) {
      const float t = fmaf(bc[0][d], dx, keep * st[i]);
      y = fmaf(t, bc[1][d], y);
      S[(uint64_t)d * V + v] = t;
    }
  }
  red[dg][col] = y;
  __syncthreads();
  if (dg == 0 && v < V) {
    y = 0.f;
#pragma unroll
    for (int i = 0; i < (int)NG; i++) y += red[i][col];
    act[s.out + (uint64_t)row * s.out_stride + h * V + v] = fmaf(skip, xv, y);
  }
  float* slot = ring + (uint64_t)(pos % s.taps) * n_ch;
  if (blockIdx.y == 0 && h % rep == 0)
    for (uint32_t d = tid; d < N; d += SSTEP) { slot[bch + d] = x[bch + d]; slot[cch + d] = x[cch + d]; }
  if (tid < VC && v0 + tid < V) slot[xch + tid] = x[xch + tid];
}

// ---- a portion ------------------------------------------------------------------------------------------------------
// Blocks of a (group, chunk): C [16][Np], B^T [Np][16], C . B [16][16]; of a (head, chunk): x [16][Vp], exp(L_t - L_s) dt_s
// [16][16], exp(L_t) [16], exp(L_last - L_s) dt_s [16].
struct SpaceDims { uint32_t Np, Vp, n_chunks; };
__host__ __device__ inline uint32_t group_floats(const SpaceDims& d) { return 32u * d.Np + 256u; }
__host__ __device__ inline uint32_t head_floats(const SpaceDims& d) { return 16u * d.Vp + 288u; }

template <int TM>
__global__ void __launch_bounds__(256)
k_space_prep(const SSpec s, const float* __restrict__ act, const float* __restrict__ state, float* __restrict__ scratch, SpaceDims sd,
             uint32_t m, uint32_t seq0, uint32_t pos) {
  extern __shared__ float lds[];
  const uint32_t N = s.state, V = s.vdim, tid = threadIdx.x, c0 = blockIdx.x * CH, inner = s.heads * V, n_ch = inner + 2u * s.groups * N;
  const float* x = act + s.x + s.x_c;
  const float* ring = state + (uint64_t)seq0 * s.seq_stride + s.conv_off;
  const auto conv = [&](uint32_t ch, auto put) {
    conv_silu_rows<TM>(x, s.x_stride, c0, m, ring, n_ch, ch, pos, act + s.conv + (uint64_t)ch * s.taps, s.taps, put, act[s.conv_b + ch]);
  };
  if (blockIdx.y < s.groups) {
    const uint32_t grp = blockIdx.y, P = N + 1u;
    float *bs = lds, *cs = lds + CH * P;
    float* oC = scratch + ((uint64_t)grp * sd.n_chunks + blockIdx.x) * group_floats(sd);
    float *oB = oC + 16u * sd.Np, *oD = oB + 16u * sd.Np;
    for (uint32_t i = tid; i < 2u * N; i += 256u) {
      const bool is_c = i >= N;
      const uint32_t d = is_c ? i - N : i;
      float* to = (is_c ? cs : bs) + d;
      conv(inner + ((is_c ? s.groups : 0u) + grp) * N + d, [&](int t, float v) { to[t * P] = v; });
    }
    __syncthreads();
    {
      const uint32_t t = tid >> 4, r = tid & 15u;
      float a = 0.f;
      if (r <= t) {
#pragma unroll 4
        for (uint32_t d = 0; d < N; d++) a = fmaf(cs[t * P + d], bs[r * P + d], a);
      }
      oD[t * 16u + r] = a;
    }
    for (uint32_t d = tid; d < sd.Np; d += 256u) {
      float b[CH];
#pragma unroll
      for (int t = 0; t < (int)CH; t++) {
        oC[t * sd.Np + d] = d < N ? cs[t * P + d] : 0.f;
        b[t] = d < N ? bs[t * P + d] : 0.f;
      }
#pragma unroll
      for (int t = 0; t < (int)CH; t += 4) *(f4_t*)(oB + d * 16u + t) = (f4_t){b[t], b[t + 1], b[t + 2], b[t + 3]};
    }
    return;
  }
  const uint32_t h = blockIdx.y - s.groups;
  float *dt = lds, *lg = lds + CH;
  float* oX = scratch + (uint64_t)s.groups * sd.n_chunks * group_floats(sd) + ((uint64_t)h * sd.n_chunks + blockIdx.x) * head_floats(sd);
  float *oM = oX + 16u * sd.Vp, *oE = oM + 256u, *oG = oE + 16u;
  if (tid < 64u) {                                            // tokens past the portion: no step, no decay
    const uint32_t t = tid & 15u;
    const bool in = c0 + t < m;
    const float d = in ? softplus_f(act[s.x + (uint64_t)(c0 + t) * s.x_stride + s.x_dt + h] + act[s.dt_bias + h]) : 0.f;
    if (tid < CH) { dt[t] = d; lg[t] = -fminf(expf(act[s.a_log + h]) * d, NO_MEMORY) * 1.44269504f; }
  }
  for (uint32_t i = tid; i < sd.Vp; i += 256u) {
    if (i < V) conv(h * V + i, [&](int t, float v) { oX[t * sd.Vp + i] = v; });
    else {
#pragma unroll
      for (int t = 0; t < (int)CH; t++) oX[t * sd.Vp + i] = 0.f;
    }
  }
  __syncthreads();
  // Decays between two tokens from the logarithms between them: the difference of two long sums would keep the rounding of
  // everything ahead of both.
  const uint32_t t = tid >> 4, r = tid & 15u;
  float l = 0.f, e = 0.f;
#pragma unroll
  for (uint32_t i = 0; i < CH; i++) { l += i > r && i <= t ? lg[i] : 0.f; e += i <= r ? lg[i] : 0.f; }
  l = r <= t ? __builtin_amdgcn_exp2f(l) * dt[r] : 0.f;
  oM[t * 16u + r] = l;
  if (t == CH - 1u) { oE[r] = __builtin_amdgcn_exp2f(e); oG[r] = l; }
}

// Four waves share the state rows (NT tiles of 16 each); a tile's accumulator holds rows 4 g + i of lane group g, which
// is also how instruction i wants its right operand when the left one is read as four consecutive columns per lane.
template <int NT> struct SpaceOps { f4_t c[NT], b[NT], cb, m, e, g; float u[4], last; };
template <int NT>
__device__ __forceinline__ void load_ops(SpaceOps<NT>& o, const float* gb, const float* hb, const SpaceDims& sd, uint32_t wave, uint32_t c,
                                         uint32_t kg, uint32_t v0) {
  const float *pB = gb + 16u * sd.Np, *pD = pB + 16u * sd.Np, *pM = hb + 16u * sd.Vp, *pE = pM + 256u, *pG = pE + 16u;
#pragma unroll
  for (int j = 0; j < NT; j++) {
    const uint32_t d0 = (wave * NT + j) * 16u;
    o.c[j] = *(const f4_t*)(gb + c * sd.Np + d0 + 4u * kg);
    o.b[j] = *(const f4_t*)(pB + (d0 + c) * 16u + 4u * kg);
  }
  o.cb = *(const f4_t*)(pD + c * 16u + 4u * kg);
  o.m = *(const f4_t*)(pM + c * 16u + 4u * kg);
  o.e = *(const f4_t*)(pE + 4u * kg);
  o.g = *(const f4_t*)(pG + 4u * kg);
  o.last = pE[15];
#pragma unroll
  for (int i = 0; i < 4; i++) o.u[i] = hb[(4u * kg + i) * sd.Vp + v0 + c];
}

template <int NT>
__global__ void __launch_bounds__(256)
k_space_scan(const SSpec s, const float* __restrict__ scratch, float* act, float* state, SpaceDims sd, uint32_t m, uint32_t seq0, uint32_t pos) {
  __shared__ f4_t pb[2][4][64];
  const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, c = lane & 15u, kg = lane >> 4;
  const uint32_t h = blockIdx.x, v0 = blockIdx.y * 16u, N = s.state, V = s.vdim, v = v0 + c, rep = s.heads / s.groups, grp = h / rep;
  const uint32_t gs = group_floats(sd), hs = head_floats(sd);
  const float* gb = scratch + (uint64_t)grp * sd.n_chunks * gs;
  const float* hb = scratch + (uint64_t)s.groups * sd.n_chunks * gs + (uint64_t)h * sd.n_chunks * hs;
  state += (uint64_t)seq0 * s.seq_stride;
  float* S = state + s.s_off + (uint64_t)h * N * V;
  const float skip = act[s.skip + h];
  f4_t st[NT];
#pragma unroll
  for (int j = 0; j < NT; j++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const uint32_t d = (wave * NT + j) * 16u + 4u * kg + i;
      st[j][i] = (pos != 0u && d < N && v < V) ? S[(uint64_t)d * V + v] : 0.f;
    }
  SpaceOps<NT> cur, nxt;
  load_ops<NT>(cur, gb, hb, sd, wave, c, kg, v0);
  for (uint32_t ci = 0; ci < sd.n_chunks; ci++) {
    if (ci + 1u < sd.n_chunks) load_ops<NT>(nxt, gb + (uint64_t)(ci + 1u) * gs, hb + (uint64_t)(ci + 1u) * hs, sd, wave, c, kg, v0);
    f4_t p = {0, 0, 0, 0};
#pragma unroll
    for (int j = 0; j < NT; j++)
#pragma unroll
      for (int i = 0; i < 4; i++) p = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.c[j][i], st[j][i], p, 0, 0, 0);
    pb[ci & 1u][wave][lane] = p;
#pragma unroll
    for (int j = 0; j < NT; j++) {
      st[j] *= cur.last;
#pragma unroll
      for (int i = 0; i < 4; i++) st[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.b[j][i], cur.g[i] * cur.u[i], st[j], 0, 0, 0);
    }
    __syncthreads();
    if (wave == (ci & 3u)) {                                  // the waves take turns with the outputs
      const f4_t* r = &pb[ci & 1u][0][0];
      f4_t o = ((r[lane] + r[64 + lane]) + (r[128 + lane] + r[192 + lane])) * cur.e;
#pragma unroll
      for (int i = 0; i < 4; i++)
        o = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.cb[i] * cur.m[i] + (c == 4u * kg + i ? skip : 0.f), cur.u[i], o, 0, 0, 0);
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const uint32_t r2 = ci * CH + 4u * kg + i;
        if (r2 < m && v < V) act[s.out + (uint64_t)r2 * s.out_stride + h * V + v] = o[i];
      }
    }
    cur = nxt;
  }
#pragma unroll
  for (int j = 0; j < NT; j++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const uint32_t d = (wave * NT + j) * 16u + 4u * kg + i;
      if (d < N && v < V) S[(uint64_t)d * V + v] = st[j][i];
    }
  const uint32_t inner = s.heads * V, n_ch = inner + 2u * s.groups * N;      // the convolution's ring
  for (uint32_t r = m > s.taps ? m - s.taps : 0u; r < m; r++) {
    float* slot = state + s.conv_off + (uint64_t)((pos + r) % s.taps) * n_ch;
    const float* x = act + s.x + s.x_c + (uint64_t)r * s.x_stride;
    if (blockIdx.y == 0 && h % rep == 0)
      for (uint32_t d = tid; d < N; d += 256u) {
        const uint32_t b = inner + grp * N + d, cc = inner + (s.groups + grp) * N + d;
        slot[b] = x[b];
        slot[cc] = x[cc];
      }
    if (wave == 0u && kg == 0u && v < V) slot[h * V + v] = x[h * V + v];
  }
}

static Scratch g_space;
void state_space_release() { scratch_free(g_space); }

}  // namespace adamah

using namespace adamah;

extern "C" int adamah_state_space_dev(uint32_t map_act, uint32_t h_spec, uint32_t n_seq, uint32_t rows, uint32_t seq0, uint32_t pos) { ADAMAH_API();
  Map* ma = get_f32_map(map_act);
  const SSpec* s = spec_of<SSpec>(h_spec);
  if (!ma || !s || n_seq == 0 || rows == 0 || (n_seq > 1 && rows > 1)) return ADAMAH_ERR_INVALID;
  Map* ms = get_f32_map(s->state_map);
  const uint64_t N = s->state, V = s->vdim, H = s->heads, G = s->groups, n_tok = (uint64_t)n_seq * rows;
  if (!ms || N == 0 || N > 256 || V == 0 || V > 256 || H == 0 || G == 0 || H % G || s->taps == 0 || s->taps > MAX_TAPS) return ADAMAH_ERR_INVALID;
  const uint64_t n_ch = H * V + 2 * G * N;
  if (s->x_c + n_ch > s->x_stride || s->x_dt + H > s->x_stride || H + G > 65535) return ADAMAH_ERR_INVALID;
  if (!in_range(s->x, n_tok * s->x_stride, ma->n_elems) || !in_range(s->out, (n_tok - 1) * s->out_stride + H * V, ma->n_elems)) return ADAMAH_ERR_INVALID;
  if (!in_range(s->conv, n_ch * s->taps, ma->n_elems) || !in_range(s->conv_b, n_ch, ma->n_elems) || !in_range(s->dt_bias, H, ma->n_elems) ||
      !in_range(s->a_log, H, ma->n_elems) || !in_range(s->skip, H, ma->n_elems)) return ADAMAH_ERR_INVALID;
  if ((uint64_t)s->s_off + H * N * V > s->seq_stride || (uint64_t)s->conv_off + n_ch * s->taps > s->seq_stride ||
      !in_range((uint64_t)seq0 * s->seq_stride, (uint64_t)n_seq * s->seq_stride, ms->n_elems)) return ADAMAH_ERR_INVALID;
  float *act = (float*)ma->buf, *state = (float*)ms->buf;
  if (rows == 1) {
    const dim3 grid((uint32_t)H, cdiv(V, VC), n_seq);
#define STEP(DN, TM) k_space_step<DN, TM><<<grid, SSTEP, 0, g.stream>>>(*s, act, state, seq0, pos)
    if (s->taps <= 4) { if (N <= 64) STEP(4, 4); else if (N <= 128) STEP(8, 4); else STEP(16, 4); }
    else { if (N <= 64) STEP(4, MAX_TAPS); else if (N <= 128) STEP(8, MAX_TAPS); else STEP(16, MAX_TAPS); }
#undef STEP
    count_launch();
    return check_launch();
  }
  const SpaceDims sd = {(uint32_t)((N + 63) / 64 * 64), (uint32_t)((V + 15) / 16 * 16), cdiv(rows, CH)};
  if (int r = scratch_need(g_space, (G * sd.n_chunks * group_floats(sd) + H * sd.n_chunks * head_floats(sd)) * 4)) return r;
  float* sc = (float*)g_space.p;
  const dim3 pg(sd.n_chunks, (uint32_t)(G + H));
  const size_t lds = std::max<size_t>(2 * CH, (size_t)2 * CH * (N + 1)) * 4;
  if (s->taps <= 4) k_space_prep<4><<<pg, 256, lds, g.stream>>>(*s, act, state, sc, sd, rows, seq0, pos);
  else k_space_prep<MAX_TAPS><<<pg, 256, lds, g.stream>>>(*s, act, state, sc, sd, rows, seq0, pos);
  count_launch();
  if (int r = check_launch()) return r;
  const dim3 grid((uint32_t)H, cdiv(V, 16));
  switch (sd.Np / 64u) {
    case 1: k_space_scan<1><<<grid, 256, 0, g.stream>>>(*s, sc, act, state, sd, rows, seq0, pos); break;
    case 2: k_space_scan<2><<<grid, 256, 0, g.stream>>>(*s, sc, act, state, sd, rows, seq0, pos); break;
    case 3: k_space_scan<3><<<grid, 256, 0, g.stream>>>(*s, sc, act, state, sd, rows, seq0, pos); break;
    default: k_space_scan<4><<<grid, 256, 0, g.stream>>>(*s, sc, act, state, sd, rows, seq0, pos); break;
  }
  count_launch();
  return check_launch();
}
