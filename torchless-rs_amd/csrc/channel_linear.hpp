// What the kernels of linear attention with a decay per key channel share: the terms of a row (see
// channel_linear.hip) and their functions.
#pragma once
#include "common.hpp"

namespace tl {

constexpr int CL_MAX_TAPS = 8;
constexpr int CL_MAX_D = 256;        // dk and dv

__device__ __forceinline__ float cl_sigmoid(float a) { return 1.0f / (1.0f + expf(-a)); }
__device__ __forceinline__ float cl_silu(float a) { return a / (1.0f + expf(-a)); }
__device__ __forceinline__ float cl_softplus(float a) { return fmaxf(a, 0.f) + log1pf(expf(-fabsf(a))); }
// log of the decay of one channel, z with its bias: rate * softplus(z), rate = -exp(A_log) of the head, or
// log(logistic(z)) * inv_tau
__device__ __forceinline__ float cl_log_decay(float z, bool rated, float rate, float inv_tau) {
  return rated ? rate * cl_softplus(z) : -cl_softplus(-z) * inv_tau;
}

// Sum over the 16 lanes of a row of a wave; every lane gets it.
__device__ __forceinline__ float row16_sum(float v) {
  v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x128, 0xf, 0xf, true));   // row_ror:8
  v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x124, 0xf, 0xf, true));   // row_ror:4
  v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x122, 0xf, 0xf, true));   // row_ror:2
  v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x121, 0xf, 0xf, true));   // row_ror:1
  return v;
}

struct ChannelTerms {
  int G, H, dk, dv;
  int b_off;                 // beta's column (-1: the plain recurrence)
  int a_off, a_rank;         // the decays' inner row
  int g_off, g_rank;         // the gate's inner row (g_rank 0: the gate is not made here)
  int taps;                  // 0: no convolution
  const float* conv_w;       // [2 G dk + H dv, taps]
  const float* bias;         // [H * dk] on the decays' z, or null
  const float* rate;         // [H]: A_log, or null: logistic(z)^(1 / tau)
  float inv_tau;
  float qscale;
  float unit_eps;            // below 0: q and k stay as they are
};

}  // namespace tl
