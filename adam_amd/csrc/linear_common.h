// Products with bfloat16 weight maps: the operand structs shared by the launchers and the ops built on them.
#pragma once
#include "common.h"
#include "../../include/adamah_hip.h"

namespace adamah {

typedef AdamahLinearSpec LinSpec;
typedef __bf16 bf16_t;
typedef bf16_t bf8_t __attribute__((ext_vector_type(8)));
typedef bf16_t bf4_t __attribute__((ext_vector_type(4)));
typedef float f4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float bf_lo(uint32_t w) { return __uint_as_float(w << 16); }
__device__ __forceinline__ float bf_hi(uint32_t w) { return __uint_as_float(w & 0xFFFF0000u); }

// sum over a row of 16 lanes, in all of them (lane permutations of the vector unit, no LDS)
__device__ __forceinline__ float row16_sum(float v) {
#define ROW16_ADD(ctrl) v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), ctrl, 0xF, 0xF, false))
  ROW16_ADD(0xB1); ROW16_ADD(0x4E); ROW16_ADD(0x141); ROW16_ADD(0x140);   // quads, then the row's halves and the row mirrored
#undef ROW16_ADD
  return v;
}

__device__ __forceinline__ float wsum64(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}

// ---- tiles of the many-row products ---------------------------------------------------------------------------------
// BM tokens x BN matrix rows, 64 columns of K a step, four waves as 2 x 2.  Tiles go straight to LDS (16 bytes a lane,
// eight rows of 128 bytes an instruction); chunk j of a row sits at slot j ^ (row & 7), which spreads the 16-byte reads
// of 16 rows over the banks.  Two buffers: the next step's loads run under this step's products.  Where a lane's rows
// start is settled once, so they may lie anywhere.
template <int R> struct TileRows {
  const bf16_t* p[R / 32];
  template <class Row>
  __device__ __forceinline__ TileRows(uint32_t wave, uint32_t lane, Row row) {
#pragma unroll
    for (int i = 0; i < R / 32; i++) {
      const uint32_t r = (uint32_t)i * 32u + wave * 8u + (lane >> 3);
      p[i] = row(r) + (((lane & 7u) ^ (r & 7u)) << 3);
    }
  }
  __device__ __forceinline__ void load(uint32_t k, bf16_t* lds, uint32_t wave) const {
#pragma unroll
    for (int i = 0; i < R / 32; i++)
      __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(p[i] + k),
                                       (__attribute__((address_space(3))) void*)(lds + ((uint32_t)i * 32u + wave * 8u) * 64u), 16, 0, 0);
  }
};
// acc[i][j]: matrix rows wn + 16 i, tokens wm + 16 j of the tile; la: 2 BN 64, lb: 2 BM 64 elements
template <int BM, int BN>
__device__ __forceinline__ void tile_product(f4_t (&acc)[BN / 32][BM / 32], const TileRows<BN>& w, const TileRows<BM>& x, uint32_t kp,
                                             bf16_t* la, bf16_t* lb, uint32_t wave, uint32_t lane) {
  constexpr int NTN = BN / 32, NTM = BM / 32;
  const uint32_t c = lane & 15u, kg = lane >> 4, wn = (wave & 1u) * (BN / 2), wm = (wave >> 1) * (BM / 2);
#pragma unroll
  for (int i = 0; i < NTN; i++)
#pragma unroll
    for (int j = 0; j < NTM; j++) acc[i][j] = (f4_t){0, 0, 0, 0};
  w.load(0, la, wave);
  x.load(0, lb, wave);
  uint32_t buf = 0;
  for (uint32_t k = 0; k < kp; k += 64u, buf ^= 1u) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();                       // this step's tiles have arrived, the other buffer is no longer read
    if (k + 64u < kp) {
      w.load(k + 64u, la + (buf ^ 1u) * (BN * 64), wave);
      x.load(k + 64u, lb + (buf ^ 1u) * (BM * 64), wave);
    }
    const bf16_t *ta = la + buf * (BN * 64), *tb = lb + buf * (BM * 64);
#pragma unroll
    for (int h = 0; h < 2; h++) {
      bf8_t a[NTN], b[NTM];
#pragma unroll
      for (int i = 0; i < NTN; i++) {
        const uint32_t r = wn + 16u * i + c;
        a[i] = *(const bf8_t*)(ta + r * 64u + (((4u * h + kg) ^ (r & 7u)) << 3));
      }
#pragma unroll
      for (int j = 0; j < NTM; j++) {
        const uint32_t r = wm + 16u * j + c;
        b[j] = *(const bf8_t*)(tb + r * 64u + (((4u * h + kg) ^ (r & 7u)) << 3));
      }
#pragma unroll
      for (int i = 0; i < NTN; i++)
#pragma unroll
        for (int j = 0; j < NTM; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[i], b[j], acc[i][j], 0, 0, 0);
    }
  }
}
// The same in float32: 64 tokens x 64 matrix rows, 32 columns a step, on the float32 matrix instruction.  Within a run of
// 16 columns, instruction i takes column 4 g + i from lane group g on both sides, so a lane's operands are one 16-byte
// read.  wsrc, xsrc: this thread's row (tid / 4 of the tile) from column (tid % 4) 8 on.
__device__ __forceinline__ void tile_product_f32(f4_t (&acc)[2][2], const bf16_t* wsrc, const float* xsrc, uint32_t kp, float (*la)[36],
                                                 float (*lb)[36]) {
  const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, c = lane & 15u, kg = lane >> 4;
  const uint32_t wn = (wave & 1u) * 32u, wm = (wave >> 1) * 32u, lr = tid >> 2, lc = (tid & 3u) * 8u;
#pragma unroll
  for (int i = 0; i < 2; i++)
#pragma unroll
    for (int j = 0; j < 2; j++) acc[i][j] = (f4_t){0, 0, 0, 0};
  for (uint32_t k = 0; k < kp; k += 32u) {
    const uint4 w = *(const uint4*)(wsrc + k);
    const float4 x0 = *(const float4*)(xsrc + k), x1 = *(const float4*)(xsrc + k + 4);
    __syncthreads();
    *(float4*)&la[lr][lc] = make_float4(bf_lo(w.x), bf_hi(w.x), bf_lo(w.y), bf_hi(w.y));
    *(float4*)&la[lr][lc + 4] = make_float4(bf_lo(w.z), bf_hi(w.z), bf_lo(w.w), bf_hi(w.w));
    *(float4*)&lb[lr][lc] = x0;
    *(float4*)&lb[lr][lc + 4] = x1;
    __syncthreads();
#pragma unroll
    for (int h = 0; h < 2; h++) {
      f4_t a[2], b[2];
#pragma unroll
      for (int i = 0; i < 2; i++) {
        a[i] = *(const f4_t*)&la[wn + 16u * i + c][16u * h + 4u * kg];
        b[i] = *(const f4_t*)&lb[wm + 16u * i + c][16u * h + 4u * kg];
      }
#pragma unroll
      for (int t = 0; t < 4; t++)
#pragma unroll
        for (int i = 0; i < 2; i++)
#pragma unroll
          for (int j = 0; j < 2; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i][t], b[j][t], acc[i][j], 0, 0, 0);
    }
  }
}

// The host copy of a spec handle, or nullptr when the handle is missing, too short or written by the device.
template <class S> inline const S* spec_of(uint32_t h) { return (const S*)res_host(h, sizeof(S) / 4); }

// Device-side growable scratch of one user; contents are only valid between launches of one op.
struct Scratch { uint8_t* p = nullptr; size_t cap = 0; };
int scratch_need(Scratch& s, size_t bytes);      // linear_bf16.hip: ADAMAH_OK or an error; never shrinks
void scratch_free(Scratch& s);

// linear_bf16.hip
int run_linear(Map* ma, Map* mo, Map* mw, const LinSpec& s, const uint32_t* row_idx, uint32_t rows);

}  // namespace adamah
