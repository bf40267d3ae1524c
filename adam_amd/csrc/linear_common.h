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

// The host copy of a spec handle, or nullptr when the handle is missing, too short or written by the device.
template <class S> inline const S* spec_of(uint32_t h) { return (const S*)res_host(h, sizeof(S) / 4); }

// Device-side growable scratch of one user; contents are only valid between launches of one op.
struct Scratch { uint8_t* p = nullptr; size_t cap = 0; };
int scratch_need(Scratch& s, size_t bytes);      // linear_bf16.hip: ADAMAH_OK or an error; never shrinks
void scratch_free(Scratch& s);

// linear_bf16.hip
int run_linear(Map* ma, Map* mo, Map* mw, const LinSpec& s, const uint32_t* row_idx, uint32_t rows);

}  // namespace adamah
