// Retention: linear attention with a fixed decay per head, no softmax and no denominator.
//
// A row of the fused projection is [q (H*dk) | k (H*dk) | v (H*dv) | g (H*dv)] in float.  q and k
// are rotated by position (the first channels of every head, pairs as `Rotation` says), k is
// multiplied by `kscale` afterwards; head h keeps a state S [dk, dv]:
//
//   S <- decay[h] S + k v^T ;   o = S^T q
//
// and the row's result is rms_head(o) * silu(g): each head's o divided by its own root mean square
// over the dv channels, no weight.  The state lives in a block per sequence, [H][dk][dv] float, and
// is carried from step to step.
//
// `retention_scan` goes row after row with everything in float: the kernel of the 32-bit path, of
// single tokens and of short portions.  Many rows in bfloat16 go by chunks on the matrix cores
// (the kernels below it).
#include "common.hpp"

namespace tl {

constexpr int RN_MAX_DK = 512;

// One workgroup per (tile of TC columns of the state, head, sequence); QN = TC / VEC lanes share a
// row of the tile, RG = 256 / QN groups of lanes go round the rows: lane (rg, quad) keeps rows rg,
// rg + RG, ... (R at most) of its VEC columns in registers.  Rows of the sequence are staged TB at a
// time; the groups' shares of a row's sums meet in LDS once a batch.
template <int R, int VEC>
__global__ void __launch_bounds__(256)
retention_scan_kernel(const float* __restrict__ proj, int width, int H, int dk, int dv, int TC, int TB,
                      const int* __restrict__ row_pos, Rotation rot, float kscale, const float* __restrict__ decay,
                      float* __restrict__ state, long long stride, const int* __restrict__ cu_seqlens,
                      const int* __restrict__ slots, float* __restrict__ o) {
  extern __shared__ __attribute__((aligned(16))) float rn_lds[];
  const int QN = TC / VEC, RG = 256 / QN, NP = R * RG;           // NP >= dk: zeros behind the dk rows
  float* qs = rn_lds;                  // [TB][NP]
  float* ks = qs + TB * NP;            // [TB][NP]
  float* vs = ks + TB * NP;            // [TB][TC]
  float* part = vs + TB * TC;          // [TB][RG][TC]
  const int c0 = blockIdx.x * TC, h = blockIdx.y, b = blockIdx.z;
  const int t = threadIdx.x, quad = t % QN, rg = t / QN;
  const int row0 = cu_seqlens[b], n_new = cu_seqlens[b + 1] - row0;
  if (n_new == 0) return;
  const int col = c0 + quad * VEC;
  const bool active = col < dv;                                  // (VEC divides dv)
  float* S_g = state + (long long)slots[b] * stride + (size_t)h * dk * dv + col;
  float S[R][VEC];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int i = rg + r * RG;
    if (active && i < dk) {
      if constexpr (VEC == 4) {
        const f32x4 w = *reinterpret_cast<const f32x4*>(S_g + (size_t)i * dv);
#pragma unroll
        for (int c = 0; c < 4; ++c) S[r][c] = w[c];
      } else {
        S[r][0] = S_g[(size_t)i * dv];
      }
    } else {
#pragma unroll
      for (int c = 0; c < VEC; ++c) S[r][c] = 0.f;
    }
  }
  const float g = decay[h];
  const int half = rot.rotary_dim / 2;
  for (int e = t; e < 2 * TB * NP; e += 256) qs[e] = 0.f;        // (qs and ks lie one behind the other)
  for (int i0 = 0; i0 < n_new; i0 += TB) {
    const int tb = min(TB, n_new - i0);
    __syncthreads();                   // the last batch has been read (and the zeros written)
    for (int e = t; e < tb * dk; e += 256) {
      // unit u of a row: a rotated pair (u < half) or a channel behind the rotated ones
      const int i = e / dk, u = e % dk;
      const float* qr = proj + (size_t)(row0 + i0 + i) * width + (size_t)h * dk;
      const float* kr = qr + (size_t)H * dk;
      if (u < half) {
        int a, d;
        pair_channels(u, rot.rotary_dim, rot.interleaved, a, d);
        float sn, cs, x, y;
        sincosf((float)row_pos[row0 + i0 + i] * rot.inv_freq[u], &sn, &cs);
        cs *= rot.magnitude;
        sn *= rot.magnitude;
        rotate_pair(qr[a], qr[d], cs, sn, x, y);
        qs[i * NP + a] = x;
        qs[i * NP + d] = y;
        rotate_pair(kr[a], kr[d], cs, sn, x, y);
        ks[i * NP + a] = x * kscale;
        ks[i * NP + d] = y * kscale;
      } else if (u >= 2 * half) {
        qs[i * NP + u] = qr[u];
        ks[i * NP + u] = kr[u] * kscale;
      }
    }
    for (int e = t; e < tb * TC; e += 256) {
      const int i = e / TC, c = e % TC;
      vs[e] = c0 + c < dv ? proj[(size_t)(row0 + i0 + i) * width + (size_t)2 * H * dk + (size_t)h * dv + c0 + c] : 0.f;
    }
    __syncthreads();
    for (int i = 0; i < tb; ++i) {
      float v[VEC], acc[VEC];
#pragma unroll
      for (int c = 0; c < VEC; ++c) {
        v[c] = vs[i * TC + quad * VEC + c];
        acc[c] = 0.f;
      }
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const float kv = ks[i * NP + rg + r * RG], qv = qs[i * NP + rg + r * RG];
#pragma unroll
        for (int c = 0; c < VEC; ++c) {
          S[r][c] = fmaf(g, S[r][c], kv * v[c]);
          acc[c] = fmaf(S[r][c], qv, acc[c]);
        }
      }
#pragma unroll
      for (int c = 0; c < VEC; ++c) part[(i * RG + rg) * TC + quad * VEC + c] = acc[c];
    }
    __syncthreads();
    for (int e = t; e < tb * TC; e += 256) {
      const int i = e / TC, c = e % TC;
      if (c0 + c >= dv) continue;
      const float* p = part + (size_t)i * RG * TC + c;
      float s0 = 0.f, s1 = 0.f, s2 = 0.f, s3 = 0.f;
      for (int q = 0; q < RG; q += 4) {          // (RG is a multiple of 4)
        s0 += p[q * TC];
        s1 += p[(q + 1) * TC];
        s2 += p[(q + 2) * TC];
        s3 += p[(q + 3) * TC];
      }
      o[(size_t)(row0 + i0 + i) * H * dv + (size_t)h * dv + c0 + c] = (s0 + s1) + (s2 + s3);
    }
  }
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int i = rg + r * RG;
    if (!active || i >= dk) continue;
    if constexpr (VEC == 4) {
      *reinterpret_cast<f32x4*>(S_g + (size_t)i * dv) = f32x4{S[r][0], S[r][1], S[r][2], S[r][3]};
    } else {
      S_g[(size_t)i * dv] = S[r][0];
    }
  }
}

// out[n, h, :] = factor * o / sqrt(mean(o^2) + eps) * w * (silu or logistic of g), one wave a head of a row; w (shared by
// the heads) may be null
template <typename T>
__global__ void __launch_bounds__(256)
heads_norm_gate_kernel(const float* __restrict__ o, const float* __restrict__ w, const float* __restrict__ gate, int gate_stride, int silu,
                       int H, int dv, float eps, float factor, int units, T* __restrict__ out, int out_stride) {
  const int unit = blockIdx.x * 4 + threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  if (unit >= units) return;
  const int n = unit / H, h = unit % H;
  const float* row = o + ((size_t)n * H + h) * dv;
  const float* gr = gate + (size_t)n * gate_stride + (size_t)h * dv;
  float ss = 0.f;
  for (int c = lane; c < dv; c += WAVE) ss += row[c] * row[c];
  const float f = factor / sqrtf(wave_sum(ss) / (float)dv + eps);
  for (int c = lane; c < dv; c += WAVE) {
    const float a = gr[c];
    out[(size_t)n * out_stride + (size_t)h * dv + c] =
        from_f32<T>(row[c] * f * (w ? w[c] : 1.f) * ((silu ? a : 1.0f) / (1.0f + expf(-a))));
  }
}

}  // namespace tl

using namespace tl;

// Columns of the state a workgroup takes: few (heads x sequences) take narrow tiles, so that every compute unit has work.
struct RetentionShape {
  int VEC, TC, RG, R, TB;
};
static RetentionShape retention_shape(int dk, int dv, long long units) {
  RetentionShape z{dv % 4 == 0 ? 4 : 1, 16, 0, 0, dk <= 256 ? 8 : 4};
  if (z.VEC == 4)
    for (int tc = 64; tc >= 16; tc /= 2) {
      z.TC = tc;
      if (units * ((dv + tc - 1) / tc) >= 512) break;
    }
  z.RG = 256 / (z.TC / z.VEC);
  z.R = (dk + z.RG - 1) / z.RG;
  int r = 1;
  while (r < z.R) r *= 2;
  z.R = r;
  return z;
}

extern "C" {

int tl_retention_scan(const float* proj, int width, int H, int dk, int dv, const int* row_pos, const float* inv_freq,
                      int rotary_dim, int interleaved, float magnitude, float kscale, const float* decay, float* state,
                      long long stride, const int* cu_seqlens, const int* slots, int n, int B, float* o, hipStream_t st) {
  TL_REQUIRE(n >= 0 && B >= 0 && H > 0 && dk > 0 && dv > 0 && dk <= RN_MAX_DK, "retention: bad sizes n=%d H=%d dk=%d dv=%d (keys up to %d)",
             n, H, dk, dv, RN_MAX_DK);
  TL_REQUIRE(width >= 2 * H * (dk + dv), "retention: a row of %d is too short for %d heads of %d/%d", width, H, dk, dv);
  TL_REQUIRE(rotary_dim >= 0 && rotary_dim % 2 == 0 && rotary_dim <= dk && (rotary_dim == 0 || inv_freq),
             "retention: %d rotated channels of a head of %d", rotary_dim, dk);
  TL_REQUIRE(proj && row_pos && decay && state && cu_seqlens && slots && o, "retention: a buffer is missing");
  TL_REQUIRE(stride >= (long long)H * dk * dv, "retention: a sequence's block is too small");
  TL_REQUIRE(H <= 65535 && B <= 65535, "retention: too many heads or sequences");
  if (n == 0 || B == 0) return 0;
  RetentionShape z = retention_shape(dk, dv, (long long)H * B);
  TL_REQUIRE(z.VEC == 1 || (stride % 4 == 0 && (uintptr_t)state % 16 == 0), "retention: a block off 16 bytes");
  const Rotation rot{inv_freq, rotary_dim, interleaved, magnitude};
  const dim3 grid((dv + z.TC - 1) / z.TC, H, B);
  const size_t lds = sizeof(float) * (size_t)z.TB * (2 * z.R * z.RG + z.TC + z.RG * z.TC);
#define TL_RN(RR, VV)                                                                                                     \
  retention_scan_kernel<RR, VV><<<grid, 256, lds, st>>>(proj, width, H, dk, dv, z.TC, z.TB, row_pos, rot, kscale, decay, \
                                                        state, stride, cu_seqlens, slots, o)
  if (z.VEC == 4) {
    if (z.R <= 1) TL_RN(1, 4);
    else if (z.R <= 2) TL_RN(2, 4);
    else if (z.R <= 4) TL_RN(4, 4);
    else if (z.R <= 8) TL_RN(8, 4);
    else if (z.R <= 16) TL_RN(16, 4);
    else TL_RN(32, 4);
  } else {
    if (z.R <= 1) TL_RN(1, 1);
    else if (z.R <= 2) TL_RN(2, 1);
    else if (z.R <= 4) TL_RN(4, 1);
    else if (z.R <= 8) TL_RN(8, 1);
    else if (z.R <= 16) TL_RN(16, 1);
    else TL_RN(32, 1);
  }
#undef TL_RN
  TL_LAUNCH_CHECK("retention_scan");
  return 0;
}

// o float [n, H*dv]; gate: the column of the first gate channel in a row of `gate_stride` floats; w [dv] or null
int tl_heads_norm_gate(const float* o, const float* w, const float* gate, int gate_stride, int silu, int n, int H, int dv, float eps,
                       float factor, void* out, int out_stride, int dt, hipStream_t st) {
  TL_REQUIRE(n >= 0 && H > 0 && dv > 0 && gate_stride >= H * dv && out_stride >= H * dv, "heads_norm_gate: bad sizes n=%d H=%d dv=%d", n, H, dv);
  TL_REQUIRE(o && gate && out, "heads_norm_gate: a buffer is missing");
  TL_REQUIRE((long long)n * H < 2147483647LL, "heads_norm_gate: too many heads");
  TL_REQUIRE(dt == DT_F32 || dt == DT_BF16, "heads_norm_gate: unknown dtype code %d", dt);
  if (n == 0) return 0;
  const int units = n * H;
  if (dt == DT_F32)
    heads_norm_gate_kernel<float><<<(units + 3) / 4, 256, 0, st>>>(o, w, gate, gate_stride, silu, H, dv, eps, factor, units, (float*)out,
                                                                  out_stride);
  else
    heads_norm_gate_kernel<bf16><<<(units + 3) / 4, 256, 0, st>>>(o, w, gate, gate_stride, silu, H, dv, eps, factor, units, (bf16*)out,
                                                                 out_stride);
  TL_LAUNCH_CHECK("heads_norm_gate");
  return 0;
}

}  // extern "C"
