// Linear attention with a decay per key channel, plain or by the delta rule.
//
// Head h keeps a state S [dk, dv]; a row brings q, k [dk], v [dv] and a decay g [dk] per channel:
//
//   plain:       S <- diag(g) S + k v^T ;                                            o = S^T q
//   delta rule:  S <- diag(g) S ;  u = beta (v - S^T k) ;  S <- S + k u^T ;          o = S^T q
//
// and the row's result is rms_head(o) * w * gate: each head's o divided by its own root mean square
// over the dv channels, times a weight that all heads share, times silu or the logistic function of
// a gate.  All of it is float.  Heads share q and k in groups: head h reads those of group
// h / (H / G).
//
// A row of the fused projection is [q (G*dk) | k (G*dk) | v (H*dv) | ...] in float, with, at columns
// that the caller names, beta's H numbers and the inner rows of the two-step projections of the
// decays and of the gate (W_2 (W_1 h): W_1's result lies in the row, the kernel applies W_2).
// `channel_rows` makes of it, row by row in float:
//
//   * q, k, v through a causal convolution per channel over the last `taps` rows (zeros before the
//     start of a sequence) and silu (optional);
//   * q and k divided by sqrt(sum of squares + unit_eps) per head (optional); q times `qscale`;
//   * the decays, z = W_2 a + bias: exp(-exp(rate_h) softplus(z)), or logistic(z)^(1 / tau);
//   * beta = logistic(b); the gate's second step (optional).
//
// `channel_scan` goes through a sequence's rows one after the other: the kernel of single tokens, of
// short portions and of the 32-bit path; a single token's norm and gate happen in the same kernel
// where a workgroup holds a whole head.  The state lives in a block per sequence,
// [conv: (taps-1) rows of (2 G dk + H dv) channels, the oldest first | S^T: H * dv * dk], and is
// carried from step to step.
#include "channel_linear.hpp"

namespace tl {

constexpr int CL_TB = 4;             // rows of a sequence that the scan stages at a time

// out[c] (for c of this wave's lanes) = sum_r W2[first + c, r] * a[r]
template <typename T>
__device__ __forceinline__ float second_step(const T* __restrict__ w2, size_t row, const float* __restrict__ a, int rank) {
  const T* w = w2 + row * rank;
  float s0 = 0.f, s1 = 0.f;
  int r = 0;
  if constexpr (sizeof(T) == 2) {
    if (rank % 8 == 0) {
      for (; r < rank; r += 8) {
        const bf16x8 x = *reinterpret_cast<const bf16x8*>(w + r);
#pragma unroll
        for (int i = 0; i < 8; i += 2) {
          s0 = fmaf((float)x[i], a[r + i], s0);
          s1 = fmaf((float)x[i + 1], a[r + i + 1], s1);
        }
      }
      return s0 + s1;
    }
  }
  for (; r + 1 < rank; r += 2) {
    s0 = fmaf(to_f32(w[r]), a[r], s0);
    s1 = fmaf(to_f32(w[r + 1]), a[r + 1], s1);
  }
  if (r < rank) s0 = fmaf(to_f32(w[r]), a[r], s0);
  return s0 + s1;
}

// z[c] = sum_r W2[first + c, r] * a[r] for c = lane, lane + 64, .. < count, handed to use(c, z).  LP lanes share a row's `rank`
// numbers (16-byte pieces of at most LP * 8 bfloat16), so that a wave's load takes whole lines; all LP loads go before the sums
template <int LP, typename F>
__device__ __forceinline__ void shared_steps(const bf16* __restrict__ w2, size_t first, int count, const float* __restrict__ a, int rank,
                                             int lane, F&& use) {
  constexpr int PER = WAVE / LP;
  const int j = lane % LP, at = lane / LP;                         // this lane's piece of rows at, at + PER, ..
  const bool in = j * 8 < rank;
  float x[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) x[e] = in ? a[j * 8 + e] : 0.f;
  for (int c0 = 0; c0 < count; c0 += WAVE) {
    bf16x8 v[LP];
#pragma unroll
    for (int p = 0; p < LP; ++p)
      v[p] = *reinterpret_cast<const bf16x8*>(w2 + (first + min(c0 + p * PER + at, count - 1)) * rank + (in ? j * 8 : 0));
    float mine = 0.f;
#pragma unroll
    for (int p = 0; p < LP; ++p) {
      float s = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) s = fmaf((float)v[p][e], x[e], s);
      if constexpr (LP == 16) {
        s = row16_sum(s);
      } else {
#pragma unroll
        for (int o = 1; o < LP; o *= 2) s += __shfl_xor(s, o, WAVE);
      }
      // row c0 + lane lies in pass lane / PER, with the lanes that share place lane % PER
      const float got = LP == 1 ? s : __shfl(s, (lane % PER) * LP, WAVE);
      if (lane / PER == p) mine = got;
    }
    if (c0 + lane < count) use(c0 + lane, mine);
  }
}
template <typename T, typename F>
__device__ __forceinline__ void second_steps(const T* __restrict__ w2, size_t first, int count, const float* __restrict__ a, int rank, int lane,
                                             F&& use) {
  if constexpr (sizeof(T) == 2) {
    if (rank % 8 == 0 && rank <= 128) {
      if (rank <= 16) shared_steps<2>(w2, first, count, a, rank, lane, use);
      else if (rank <= 32) shared_steps<4>(w2, first, count, a, rank, lane, use);
      else if (rank <= 64) shared_steps<8>(w2, first, count, a, rank, lane, use);
      else shared_steps<16>(w2, first, count, a, rank, lane, use);
      return;
    }
  }
  for (int c = lane; c < count; c += WAVE) use(c, second_step(w2, first + c, a, rank));
}

// One wave a unit of a row: a head of q, of k (G each), of v, of the decays (H each), of the gate (H, if made here), and
// one unit for the betas.  `single`: every sequence brings one row, and the convolution's block is shifted on the way.
template <typename T>
__global__ void __launch_bounds__(256)
channel_rows_kernel(const float* __restrict__ proj, int width, ChannelTerms t, const T* __restrict__ a2, const T* __restrict__ g2,
                    float* __restrict__ conv_state, long long stride, const int* __restrict__ row_seq,
                    const int* __restrict__ cu_seqlens, const int* __restrict__ slots, int single, float* __restrict__ q,
                    float* __restrict__ k, float* __restrict__ v, float* __restrict__ decay, float* __restrict__ beta,
                    float* __restrict__ gate) {
  const int n = blockIdx.x, lane = threadIdx.x % WAVE;
  int unit = blockIdx.y * 4 + threadIdx.x / WAVE;
  const int Q = t.G * t.dk, V = t.H * t.dv, C = 2 * Q + V;
  const float* row = proj + (size_t)n * width;
  if (unit < 2 * t.G + t.H) {                      // a head of q, k or v
    const bool is_v = unit >= 2 * t.G;
    const int d = is_v ? t.dv : t.dk;
    const int c0 = is_v ? 2 * Q + (unit - 2 * t.G) * t.dv : unit * t.dk;
    const int b = t.taps ? row_seq[n] : 0;
    const int i = t.taps ? n - cu_seqlens[b] : 0;
    float* st = t.taps ? conv_state + (long long)slots[b] * stride : nullptr;
    auto value = [&](int c) {
      if (!t.taps) return row[c];
      const float* w = t.conv_w + (size_t)c * t.taps;
      float u[CL_MAX_TAPS], wv[CL_MAX_TAPS];           // (all asked for before the block is shifted)
#pragma unroll
      for (int j = 0; j < CL_MAX_TAPS; ++j) {
        if (j >= t.taps) break;
        const int src = i - (t.taps - 1 - j);
        u[j] = src >= 0 ? row[c - (ptrdiff_t)(t.taps - 1 - j) * width] : st[(size_t)(t.taps - 1 + src) * C + c];
        wv[j] = w[j];
      }
      float acc = 0.f;
#pragma unroll
      for (int j = 0; j < CL_MAX_TAPS; ++j) {
        if (j >= t.taps) break;
        acc = fmaf(wv[j], u[j], acc);
        if (single && j > 0) st[(size_t)(j - 1) * C + c] = u[j];
      }
      return cl_silu(acc);
    };
    float x[CL_MAX_D / WAVE];
    float ss = 0.f;
#pragma unroll
    for (int r = 0; r < CL_MAX_D / WAVE; ++r) {
      const int c = lane + r * WAVE;
      x[r] = c < d ? value(c0 + c) : 0.f;
      ss += x[r] * x[r];
    }
    float f = 1.f;
    if (!is_v) {
      if (t.unit_eps >= 0.f) f = 1.0f / sqrtf(wave_sum(ss) + t.unit_eps);
      if (unit < t.G) f *= t.qscale;
    }
    float* out = is_v ? v + (size_t)n * V + (c0 - 2 * Q) : (unit < t.G ? q : k) + (size_t)n * Q + (unit % t.G) * t.dk;
#pragma unroll
    for (int r = 0; r < CL_MAX_D / WAVE; ++r) {
      const int c = lane + r * WAVE;
      if (c < d) out[c] = x[r] * f;
    }
    return;
  }
  unit -= 2 * t.G + t.H;
  if (unit < t.H) {                                // a head's decays
    const float rate = t.rate ? -expf(t.rate[unit]) : 0.f;
    second_steps(a2, (size_t)unit * t.dk, t.dk, row + t.a_off, t.a_rank, lane, [&](int c, float z) {
      const int at = unit * t.dk + c;
      decay[(size_t)n * t.H * t.dk + at] = expf(cl_log_decay(z + (t.bias ? t.bias[at] : 0.f), t.rate != nullptr, rate, t.inv_tau));
    });
    return;
  }
  unit -= t.H;
  if (t.g_rank) {
    if (unit < t.H) {                              // a head's gates
      second_steps(g2, (size_t)unit * t.dv, t.dv, row + t.g_off, t.g_rank, lane,
                   [&](int c, float z) { gate[(size_t)n * V + unit * t.dv + c] = z; });
      return;
    }
    unit -= t.H;
  }
  if (unit == 0 && t.b_off >= 0)
    for (int h = lane; h < t.H; h += WAVE) beta[(size_t)n * t.H + h] = cl_sigmoid(row[t.b_off + h]);
}

// One workgroup per (part of a head's columns, head, sequence).  The state is kept column by column, S^T [dv, dk]:
// the 16 lanes of a row of a wave share DC columns, lane s the channels (r * 16 + s) * VEC + j, so that a sum over the
// channels stays within the row and a row of the sequence costs no barrier.  Rows are staged CL_TB at a time.
struct ScanOut {
  float* o;                  // [n, H * dv] float, or null: the rows are single tokens and a workgroup holds a head:
  const float* w;            // [dv] (null: no weight)
  const float* gate;         // the gate's first column in rows `gate_stride` apart
  int gate_stride, gate_silu;
  float eps, factor;
  void* out;                 // [n, ..] in the compute dtype, rows `out_stride` apart
  int out_stride, out_f32;
};

template <int R, int VEC, int DC, bool DELTA>
__global__ void __launch_bounds__(512)
channel_scan_kernel(const float* __restrict__ q, const float* __restrict__ k, const float* __restrict__ v,
                    const float* __restrict__ decay, const float* __restrict__ beta, int G, int H, int dk, int dv,
                    float* __restrict__ state, long long stride, const int* __restrict__ cu_seqlens,
                    const int* __restrict__ slots, ScanOut z) {
  constexpr int NP = 16 * R * VEC;                               // at least dk: zeros behind the dk channels
  extern __shared__ __attribute__((aligned(16))) float cl_lds[];
  const int groups = blockDim.x / 16, TC = groups * DC;
  float* qs = cl_lds;                  // [CL_TB][NP]
  float* ks = qs + CL_TB * NP;
  float* gs = ks + CL_TB * NP;
  float* vs = gs + CL_TB * NP;         // [CL_TB][TC]
  float* os = vs + CL_TB * TC;         // [CL_TB][TC]
  float* bs = os + CL_TB * TC;         // [CL_TB]
  float* sh = bs + CL_TB;              // [blockDim.x / WAVE]
  const int c0 = blockIdx.x * TC, h = blockIdx.y, b = blockIdx.z;
  const int t = threadIdx.x, s = t % 16, cg = t / 16, NT = blockDim.x;
  const int row0 = cu_seqlens[b], n_new = cu_seqlens[b + 1] - row0;
  if (n_new == 0) return;
  const int kh = h / (H / G);
  float* S_g = state + (long long)slots[b] * stride + ((size_t)h * dv + c0 + cg * DC) * dk;
  // a single token's gate (and the norm's weight), asked for before anything waits
  constexpr int GC = 2;                                          // columns of a head a thread, at most
  float gt[GC], wt[GC];
  if (!z.o) {
#pragma unroll
    for (int r = 0; r < GC; ++r) {
      const int c = threadIdx.x + r * blockDim.x;
      gt[r] = c < dv ? z.gate[(size_t)row0 * z.gate_stride + (size_t)h * dv + c] : 0.f;
      wt[r] = c < dv && z.w ? z.w[c] : 1.f;
    }
  }
  float S[DC][R * VEC];
#pragma unroll
  for (int c = 0; c < DC; ++c)
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int d = (r * 16 + s) * VEC;
      const bool in = c0 + cg * DC + c < dv && d < dk;           // (VEC divides dk)
      if constexpr (VEC == 4) {
        const f32x4 w = in ? *reinterpret_cast<const f32x4*>(S_g + (size_t)c * dk + d) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < 4; ++j) S[c][r * 4 + j] = w[j];
      } else {
        S[c][r] = in ? S_g[(size_t)c * dk + d] : 0.f;
      }
    }
  for (int i0 = 0; i0 < n_new; i0 += CL_TB) {
    const int tb = min(CL_TB, n_new - i0);
    __syncthreads();                   // the last batch has been read
    for (int e = t; e < tb * NP; e += NT) {
      const int i = e / NP, d = e % NP;
      const size_t row = (size_t)(row0 + i0 + i);
      const bool in = d < dk;
      qs[e] = in ? q[(row * G + kh) * dk + d] : 0.f;
      ks[e] = in ? k[(row * G + kh) * dk + d] : 0.f;
      gs[e] = in ? decay[(row * H + h) * dk + d] : 0.f;
    }
    for (int e = t; e < tb * TC; e += NT) {
      const int i = e / TC, c = c0 + e % TC;
      vs[e] = c < dv ? v[((size_t)(row0 + i0 + i) * H + h) * dv + c] : 0.f;
    }
    if (DELTA && t < tb) bs[t] = beta[(size_t)(row0 + i0 + t) * H + h];
    __syncthreads();
    for (int i = 0; i < tb; ++i) {
      float u[DC], acc[DC];
      float kr[R * VEC];
#pragma unroll
      for (int c = 0; c < DC; ++c) {
        u[c] = vs[i * TC + cg * DC + c];
        acc[c] = 0.f;
      }
#pragma unroll
      for (int r = 0; r < R; ++r)
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          const int at = i * NP + (r * 16 + s) * VEC + j;
          const float g = gs[at];
          kr[r * VEC + j] = ks[at];
#pragma unroll
          for (int c = 0; c < DC; ++c) {
            S[c][r * VEC + j] *= g;
            if constexpr (DELTA) acc[c] = fmaf(S[c][r * VEC + j], kr[r * VEC + j], acc[c]);
          }
        }
      if constexpr (DELTA) {
        const float bt = bs[i];
#pragma unroll
        for (int c = 0; c < DC; ++c) {
          u[c] = bt * (u[c] - row16_sum(acc[c]));
          acc[c] = 0.f;
        }
      }
#pragma unroll
      for (int r = 0; r < R; ++r)
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          const float qv = qs[i * NP + (r * 16 + s) * VEC + j];
#pragma unroll
          for (int c = 0; c < DC; ++c) {
            S[c][r * VEC + j] = fmaf(kr[r * VEC + j], u[c], S[c][r * VEC + j]);
            acc[c] = fmaf(S[c][r * VEC + j], qv, acc[c]);
          }
        }
#pragma unroll
      for (int c = 0; c < DC; ++c) {
        const float sum = row16_sum(acc[c]);
        if (s == c % 16) os[i * TC + cg * DC + c] = sum;
      }
    }
    __syncthreads();
    if (z.o) {
      for (int e = t; e < tb * TC; e += NT) {
        const int i = e / TC, c = c0 + e % TC;
        if (c < dv) z.o[((size_t)(row0 + i0 + i) * H + h) * dv + c] = os[e];
      }
    }
  }
#pragma unroll
  for (int c = 0; c < DC; ++c)
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int d = (r * 16 + s) * VEC;
      if (c0 + cg * DC + c >= dv || d >= dk) continue;
      if constexpr (VEC == 4)
        *reinterpret_cast<f32x4*>(S_g + (size_t)c * dk + d) = f32x4{S[c][r * 4], S[c][r * 4 + 1], S[c][r * 4 + 2], S[c][r * 4 + 3]};
      else
        S_g[(size_t)c * dk + d] = S[c][r];
    }
  if (z.o) return;
  // a single token, all columns of the head here: the norm over the head and the gate
  float ss = 0.f;
  for (int c = t; c < dv; c += NT) ss += os[c] * os[c];
  ss = wave_sum(ss);
  if (t % WAVE == 0) sh[t / WAVE] = ss;
  __syncthreads();
  float sum = 0.f;
  for (int w = 0; w < NT / WAVE; ++w) sum += sh[w];
  const float f = z.factor / sqrtf(sum / (float)dv + z.eps);
#pragma unroll
  for (int r = 0; r < GC; ++r) {
    const int c = t + r * NT;
    if (c >= dv) break;
    const float a = os[c] * f * wt[r] * (z.gate_silu ? cl_silu(gt[r]) : cl_sigmoid(gt[r]));
    const size_t at = (size_t)row0 * z.out_stride + (size_t)h * dv + c;
    if (z.out_f32) ((float*)z.out)[at] = a;
    else ((bf16*)z.out)[at] = (bf16)a;
  }
}

template <int R, int VEC, int DC>
static void scan_by_rule(bool delta, dim3 grid, int threads, size_t lds, hipStream_t st, const float* q, const float* k, const float* v,
                         const float* decay, const float* beta, int G, int H, int dk, int dv, float* state, long long stride,
                         const int* cu, const int* slots, const ScanOut& z) {
  if (delta)
    channel_scan_kernel<R, VEC, DC, true><<<grid, threads, lds, st>>>(q, k, v, decay, beta, G, H, dk, dv, state, stride, cu, slots, z);
  else
    channel_scan_kernel<R, VEC, DC, false><<<grid, threads, lds, st>>>(q, k, v, decay, beta, G, H, dk, dv, state, stride, cu, slots, z);
}

}  // namespace tl

using namespace tl;

extern "C" {

// proj [n, width] float: q at column 0, k and v behind it.  a2 [H*dk, a_rank] and g2 [H*dv, g_rank] of dtype `w_dt`.
// conv_w [2 G dk + H dv, taps] float with conv_state [slots] blocks `stride` floats apart, or taps 0.
int tl_channel_rows(const float* proj, int width, int G, int H, int dk, int dv, int b_off, int a_off, int a_rank, int g_off, int g_rank,
                    int taps, const float* conv_w, const float* bias, const float* rate, float inv_tau, float qscale, float unit_eps,
                    const void* a2, const void* g2, int w_dt, float* conv_state, long long stride, const int* row_seq,
                    const int* cu_seqlens, const int* slots, int n, int B, int single, float* q, float* k, float* v, float* decay,
                    float* beta, float* gate, hipStream_t st) {
  TL_REQUIRE(n >= 0 && B >= 0 && G > 0 && H > 0 && H % G == 0 && dk > 0 && dv > 0 && dk <= CL_MAX_D && dv <= CL_MAX_D,
             "channel_rows: bad sizes n=%d G=%d H=%d dk=%d dv=%d (heads up to %d)", n, G, H, dk, dv, CL_MAX_D);
  const int C = 2 * G * dk + H * dv;
  TL_REQUIRE(b_off < 0 || b_off + H <= width, "channel_rows: a row of %d is too short", width);
  TL_REQUIRE(C <= width && a_rank > 0 && a_off >= 0 && a_off + a_rank <= width && g_rank >= 0 && (g_rank == 0 || (g_off >= 0 && g_off + g_rank <= width)),
             "channel_rows: a row of %d does not hold the inner rows of %d and %d", width, a_rank, g_rank);
  TL_REQUIRE(taps >= 0 && taps <= CL_MAX_TAPS, "channel_rows: %d taps (up to %d)", taps, CL_MAX_TAPS);
  TL_REQUIRE(taps == 0 || (conv_w && (conv_state || taps == 1) && row_seq && cu_seqlens && slots && stride >= (long long)(taps - 1) * C),
             "channel_rows: a convolution without weights, or a block too small for %d rows of %d", taps - 1, C);
  TL_REQUIRE(proj && a2 && q && k && v && decay && (b_off < 0 || beta) && (g_rank == 0 || (g2 && gate)), "channel_rows: a buffer is missing");
  TL_REQUIRE(!single || n == B, "channel_rows: %d rows of %d sequences are not one row each", n, B);
  TL_REQUIRE((uintptr_t)a2 % 16 == 0 && (uintptr_t)g2 % 16 == 0, "channel_rows: a matrix off 16 bytes");
  TL_REQUIRE(w_dt == DT_F32 || w_dt == DT_BF16, "channel_rows: unknown dtype code %d", w_dt);
  if (n == 0 || B == 0) return 0;
  const ChannelTerms t{G, H, dk, dv, b_off, a_off, a_rank, g_off, g_rank, taps, conv_w, bias, rate, inv_tau, qscale, unit_eps};
  const int units = 2 * G + 2 * H + (g_rank ? H : 0) + 1;
  const dim3 grid(n, (units + 3) / 4);
  if (w_dt == DT_F32)
    channel_rows_kernel<float><<<grid, 256, 0, st>>>(proj, width, t, (const float*)a2, (const float*)g2, conv_state, stride, row_seq,
                                                     cu_seqlens, slots, single, q, k, v, decay, beta, gate);
  else
    channel_rows_kernel<bf16><<<grid, 256, 0, st>>>(proj, width, t, (const bf16*)a2, (const bf16*)g2, conv_state, stride, row_seq,
                                                    cu_seqlens, slots, single, q, k, v, decay, beta, gate);
  TL_LAUNCH_CHECK("channel_rows");
  return 0;
}

// May a single token's norm and gate be done by the scan (one workgroup holds a head)?
int tl_channel_scan_whole(int dk, int dv) { return dv <= CL_MAX_D && dk <= CL_MAX_D ? 1 : 0; }

// o float [n, H*dv]; or o null: every sequence brings one row, and out [n, ..] = factor * rms(o) * w * (silu or logistic of gate).
int tl_channel_scan(const float* q, const float* k, const float* v, const float* decay, const float* beta, int G, int H, int dk,
                    int dv, float* state, long long stride, const int* cu_seqlens, const int* slots, int n, int B, float* o,
                    const float* w, const float* gate, int gate_stride, int gate_silu, float eps, float factor, void* out,
                    int out_stride, int out_dt, hipStream_t st) {
  TL_REQUIRE(n >= 0 && B >= 0 && G > 0 && H > 0 && H % G == 0 && dk > 0 && dv > 0 && dk <= CL_MAX_D && dv <= CL_MAX_D,
             "channel_scan: bad sizes n=%d G=%d H=%d dk=%d dv=%d (heads up to %d)", n, G, H, dk, dv, CL_MAX_D);
  TL_REQUIRE(q && k && v && decay && state && cu_seqlens && slots, "channel_scan: a buffer is missing");
  TL_REQUIRE(o || (gate && out && n == B && gate_stride >= H * dv && out_stride >= H * dv && (out_dt == DT_F32 || out_dt == DT_BF16)),
             "channel_scan: the norm and the gate need single tokens, a gate and a result");
  TL_REQUIRE(stride >= (long long)H * dk * dv, "channel_scan: a sequence's block is too small");
  TL_REQUIRE(H <= 65535 && B <= 65535, "channel_scan: too many heads or sequences");
  if (n == 0 || B == 0) return 0;
  const bool vec = dk % 4 == 0 && stride % 4 == 0 && (uintptr_t)state % 16 == 0;
  const int VEC = vec ? 4 : 1;
  int R = vec ? 1 : 2;
  while (16 * R * VEC < dk) R *= 2;
  // columns a lane's row of 16 takes, and threads: a whole head for a single token with norm and gate, else narrow
  // parts, so that every compute unit has work
  int DC = 1, threads = 256;
  if (!o) {
    if (dv > 64) threads = 512;
    while ((threads / 16) * DC < dv) DC *= 2;                  // (dv up to 256: 8 columns)
  } else {
    const long long units = (long long)H * B;
    while (DC < 4 && (256 / 16) * DC < dv && units * ((dv + 32 * DC - 1) / (32 * DC)) >= 512) DC *= 2;
  }
  const int TC = threads / 16 * DC, NP = 16 * R * VEC;
  const dim3 grid((dv + TC - 1) / TC, H, B);
  TL_REQUIRE(o || grid.x == 1, "channel_scan: a head of %d columns does not fit a workgroup", dv);
  const size_t lds = sizeof(float) * ((size_t)CL_TB * (3 * NP + 2 * TC + 1) + threads / WAVE);
  const ScanOut z{o, w, gate, gate_stride, gate_silu, eps, factor, out, out_stride, out_dt == DT_F32};
  const bool delta = beta != nullptr;
#define TL_CS(RR, VV, DD) \
  scan_by_rule<RR, VV, DD>(delta, grid, threads, lds, st, q, k, v, decay, beta, G, H, dk, dv, state, stride, cu_seqlens, slots, z)
#define TL_CSD(RR, VV)              \
  do {                              \
    if (DC == 1) TL_CS(RR, VV, 1);  \
    else if (DC == 2) TL_CS(RR, VV, 2); \
    else if (DC == 4) TL_CS(RR, VV, 4); \
    else TL_CS(RR, VV, 8);          \
  } while (0)
  if (vec) {
    if (R == 1) TL_CSD(1, 4);
    else if (R == 2) TL_CSD(2, 4);
    else TL_CSD(4, 4);
  } else {
    if (R <= 2) TL_CSD(2, 1);
    else if (R <= 4) TL_CSD(4, 1);
    else if (R <= 8) TL_CSD(8, 1);
    else TL_CSD(16, 1);
  }
#undef TL_CSD
#undef TL_CS
  TL_LAUNCH_CHECK("channel_scan");
  return 0;
}

}  // extern "C"
