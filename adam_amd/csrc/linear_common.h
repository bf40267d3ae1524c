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

// The host copy of a spec handle, or nullptr when the handle is missing, too short or written by the device.
template <class S> inline const S* spec_of(uint32_t h) { return (const S*)res_host(h, sizeof(S) / 4); }

// Device-side growable scratch of one user; contents are only valid between launches of one op.
struct Scratch { uint8_t* p = nullptr; size_t cap = 0; };
int scratch_need(Scratch& s, size_t bytes);      // linear_bf16.hip: ADAMAH_OK or an error; never shrinks
void scratch_free(Scratch& s);

// linear_bf16.hip
int run_linear(Map* ma, Map* mo, Map* mw, const LinSpec& s, const uint32_t* row_idx, uint32_t rows);

}  // namespace adamah
