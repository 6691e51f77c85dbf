// A routed mixture of small feed-forward layers ("experts").
//
// Router, per row, in float: z = W_r h (+ bias), s = softmax(z) over all E experts (or, `logistic`, every
// expert's own 1 / (1 + exp(-z))).  The choice goes by c = s, or c = s + correction[e] (which may be
// negative).  The experts form `groups` equal groups of neighbours; a group's score is its largest
// c, or the sum of its two largest (`two_largest`), and only experts of the `keep` best groups can be
// chosen (groups == 0: every expert can).  Of those the `top` with the largest c are chosen; their
// weights are their s, as they are or divided by (their sum + normalise_eps) (`normalise`).  Of equal
// scores the one with the smaller index goes first.  A shared expert may have a weight of its own, the
// logistic function of one more row of the router's matrix (`shared_weight`).
//
// `route` leaves the weights as a row of E floats, zero for an expert that was not chosen.
// The experts run as ONE wide feed-forward: the rows of all up projections stacked (the shared
// expert's behind them), the activation times the row's weight of the column's expert
// (`expert_act`), and all down projections side by side: an expert with weight zero adds nothing.
// Steps of few rows run the chosen experts alone instead (`expert_rows_up`, `expert_rows_down`).
#include "common.hpp"

namespace tl {

constexpr int RT_MAX_E = 1024;

// NT threads a row: a quarter of a thousand, or 1024 for steps of few rows, where a row's dots are what the step waits
// for (16 waves take 16 experts at a time instead of 4).  A dot is one wave's either way: the same bits.
struct RouteTerms {
  const float* correction;   // [E] or null
  int two_largest;
  int normalise;
  float normalise_eps;
  float* shared_weight;      // [n] or null; with it the router's matrix has a row E
  const float* bias;         // [E] on the products, or null
};

template <typename T, int NT>
__global__ void __launch_bounds__(NT)
route_kernel(const T* __restrict__ h, int W, const float* __restrict__ wr, int E, int groups, int keep, int top,
             int logistic, RouteTerms k, float* __restrict__ weights, int* __restrict__ chosen, bool vec) {
  __shared__ float s_s[RT_MAX_E + 1];
  __shared__ float c_s[RT_MAX_E];          // what the choice goes by
  __shared__ float g_s[RT_MAX_E];
  __shared__ unsigned char ok_s[RT_MAX_E];
  __shared__ float sh[NT / WAVE];
  const int n = blockIdx.x;
  const int t = threadIdx.x, lane = t % WAVE, wave = t / WAVE;
  const T* row = h + (size_t)n * W;
  const int rows = E + (k.shared_weight ? 1 : 0);
  for (int e = wave; e < rows; e += NT / WAVE) {
    const float* w = wr + (size_t)e * W;
    float d0 = 0.f, d1 = 0.f, d2 = 0.f, d3 = 0.f;      // four chains: the loads of one do not wait for another's sum
    int c = 0;
    if (vec) {                                         // four channels a lane and load
#pragma unroll 4
      for (c = lane * 4; c + 3 < W; c += WAVE * 4) {
        const f32x4 wv = *reinterpret_cast<const f32x4*>(w + c);
        float r0, r1, r2, r3;
        if constexpr (sizeof(T) == 2) {
          const bf16x4 rv = *reinterpret_cast<const bf16x4*>(row + c);
          r0 = (float)rv[0], r1 = (float)rv[1], r2 = (float)rv[2], r3 = (float)rv[3];
        } else {
          const f32x4 rv = *reinterpret_cast<const f32x4*>(row + c);
          r0 = rv[0], r1 = rv[1], r2 = rv[2], r3 = rv[3];
        }
        d0 = fmaf(wv[0], r0, d0);
        d1 = fmaf(wv[1], r1, d1);
        d2 = fmaf(wv[2], r2, d2);
        d3 = fmaf(wv[3], r3, d3);
      }
    } else {
      for (c = lane; c < W; c += WAVE) d0 = fmaf(w[c], to_f32(row[c]), d0);
    }
    float dot = wave_sum((d0 + d1) + (d2 + d3));
    if (lane == 0) s_s[e] = dot + (k.bias && e < E ? k.bias[e] : 0.f);
  }
  __syncthreads();
  if (k.shared_weight && t == 0) k.shared_weight[n] = 1.0f / (1.0f + expf(-s_s[E]));
  if (logistic) {                                      // every expert's score by itself
    for (int e = t; e < E; e += NT) s_s[e] = 1.0f / (1.0f + expf(-s_s[e]));
  } else {
    float m = -INFINITY;
    for (int e = t; e < E; e += NT) m = fmaxf(m, s_s[e]);
    m = block_max<NT>(m, sh);
    float sum = 0.f;
    for (int e = t; e < E; e += NT) sum += expf(s_s[e] - m);
    sum = block_sum<NT>(sum, sh);
    __syncthreads();
    for (int e = t; e < E; e += NT) s_s[e] = expf(s_s[e] - m) / sum;
  }
  __syncthreads();
  for (int e = t; e < E; e += NT) c_s[e] = s_s[e] + (k.correction ? k.correction[e] : 0.f);
  __syncthreads();
  if (groups > 0) {
    const int per = E / groups;
    for (int g = t; g < groups; g += NT) {
      float best = c_s[g * per], second = -INFINITY;
      for (int i = 1; i < per; ++i) {
        const float c = c_s[g * per + i];
        second = fmaxf(second, fminf(best, c));
        best = fmaxf(best, c);
      }
      g_s[g] = k.two_largest && per > 1 ? best + second : best;
    }
    __syncthreads();
    for (int g = t; g < groups; g += NT) {
      int ahead = 0;
      const float mine = g_s[g];
      for (int o = 0; o < groups; ++o) ahead += (g_s[o] > mine || (g_s[o] == mine && o < g)) ? 1 : 0;
      for (int i = 0; i < per; ++i) ok_s[g * per + i] = ahead < keep;
    }
  } else {
    for (int e = t; e < E; e += NT) ok_s[e] = 1;
  }
  __syncthreads();
  float mine_sum = 0.f;
  for (int e = t; e < E; e += NT) {
    float wgt = 0.f;
    if (ok_s[e]) {
      int ahead = 0;
      const float mine = c_s[e];
      for (int o = 0; o < E; ++o) ahead += (ok_s[o] && (c_s[o] > mine || (c_s[o] == mine && o < e))) ? 1 : 0;
      if (ahead < top) {
        wgt = s_s[e];
        if (chosen) chosen[(size_t)n * top + ahead] = e;
      }
    }
    if (k.normalise) {
      g_s[e] = wgt;                        // (the groups' scores have been read)
      mine_sum += wgt;
    } else {
      weights[(size_t)n * E + e] = wgt;
    }
  }
  if (k.normalise) {
    const float sum = block_sum<NT>(mine_sum, sh) + k.normalise_eps;
    for (int e = t; e < E; e += NT) weights[(size_t)n * E + e] = g_s[e] / sum;      // (a thread's own entries)
  }
}

// act = the square of max(., 0) (code 0), max(., 0) (code 1), or xIELU (code 2) with two numbers a and b:
// a z^2 + z/2 where z > 0, b (exp(z) - 1 - z) + z/2 elsewhere
struct UnaryAct {
  int code;
  float a, b;
};
__device__ __forceinline__ float unary_act(float z, const UnaryAct& k) {
  if (k.code == 2) return z > 0.f ? fmaf(k.a * z, z, 0.5f * z) : fmaf(k.b, expm1f(z) - z, 0.5f * z);
  const float r = fmaxf(z, 0.f);
  return k.code == 0 ? r * r : r;
}

// out[n, j] = act(u[n, j]) * (j < E * ff ? weights[n, j / ff] : shared_w ? shared_w[n] : 1)
template <typename T>
__global__ void __launch_bounds__(256)
expert_act_kernel(const float* __restrict__ u, const float* __restrict__ weights, const float* __restrict__ shared_w, int E,
                  int ff, int total, UnaryAct act, T* __restrict__ out) {
  const int n = blockIdx.x;
  for (int j = blockIdx.y * 256 + threadIdx.x; j < total; j += gridDim.y * 256) {
    float a = unary_act(u[(size_t)n * total + j], act);
    if (j < E * ff) a *= weights[(size_t)n * E + j / ff];
    else if (shared_w) a *= shared_w[n];
    out[(size_t)n * total + j] = from_f32<T>(a);
  }
}

// out[i] = act(u[i]) over `total` elements (a multiple of 8), u float or bfloat16: the activation of a plain feed-forward
template <typename U, typename T>
__global__ void __launch_bounds__(256)
unary_act_kernel(const U* __restrict__ u, size_t total, UnaryAct act, T* __restrict__ out) {
  for (size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * 8; i < total; i += (size_t)gridDim.x * 256 * 8) {
    float z[8];
    if constexpr (sizeof(U) == 2) {
      const bf16x8 v = *reinterpret_cast<const bf16x8*>(u + i);
#pragma unroll
      for (int e = 0; e < 8; ++e) z[e] = (float)v[e];
    } else {
      const f32x4 a = *reinterpret_cast<const f32x4*>(u + i), b = *reinterpret_cast<const f32x4*>(u + i + 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        z[e] = a[e];
        z[4 + e] = b[e];
      }
    }
    if constexpr (sizeof(T) == 2) {
      bf16x8 r;
#pragma unroll
      for (int e = 0; e < 8; ++e) r[e] = (bf16)unary_act(z[e], act);
      *reinterpret_cast<bf16x8*>(out + i) = r;
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) out[i + e] = unary_act(z[e], act);
    }
  }
}

// ---- the chosen experts alone, row by row ---------------------------------------------------------------
// For steps of few rows (fewer chosen experts than there are experts) the wide feed-forward would read every
// expert's weights to use a few: here a row reads the weights of its own `top` experts and of the shared one,
// as two products of a matrix with a vector each.  up [E * ff + shared, H] and down [H, E * ff + shared] are
// the stacked matrices of the wide form, row-major.  Slot k < top of row n is expert chosen[n, k] with the
// router's weight, slot `top` (with a shared expert) is the shared one with weight 1.

// sum_i a[i] * b[i] over one wave; `vec`: both rows are aligned for loads of 16 bytes and len is a multiple of
// the vector's length
template <typename T>
__device__ __forceinline__ float wave_dot(const T* __restrict__ a, const T* __restrict__ b, int len, bool vec, int lane) {
  float acc = 0.f;
  if (vec) {
    if constexpr (sizeof(T) == 2) {
      for (int i = lane * 8; i < len; i += WAVE * 8) {
        const bf16x8 x = *reinterpret_cast<const bf16x8*>(a + i);
        const bf16x8 y = *reinterpret_cast<const bf16x8*>(b + i);
#pragma unroll
        for (int j = 0; j < 8; ++j) acc = fmaf((float)x[j], (float)y[j], acc);
      }
    } else {
      for (int i = lane * 4; i < len; i += WAVE * 4) {
        const f32x4 x = *reinterpret_cast<const f32x4*>(a + i);
        const f32x4 y = *reinterpret_cast<const f32x4*>(b + i);
#pragma unroll
        for (int j = 0; j < 4; ++j) acc = fmaf(x[j], y[j], acc);
      }
    }
  } else {
    for (int i = lane; i < len; i += WAVE) acc = fmaf(to_f32(a[i]), to_f32(b[i]), acc);
  }
  return wave_sum(acc);
}

constexpr int ER_ROWS = 16;      // outputs of a workgroup: four a wave

// hs[n, k * ff + j] = act(up[e_k * ff + j] . y[n]) * s[n, e_k];  hs[n, top * ff + j] = act(up[E * ff + j] . y[n])
template <typename T>
__global__ void __launch_bounds__(256)
expert_rows_up_kernel(const T* __restrict__ y, int H, const T* __restrict__ up, const int* __restrict__ chosen,
                      const float* __restrict__ weights, const float* __restrict__ shared_w, int E, int top, int ff, int shared,
                      UnaryAct act, bool vec, T* __restrict__ hs) {
  const int slots = top + (shared ? 1 : 0);
  const int n = blockIdx.x / slots, k = blockIdx.x % slots;
  const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
  int base, count;
  float scale = 1.f;
  if (k < top) {
    const int e = chosen[(size_t)n * top + k];
    base = e * ff;
    count = ff;
    scale = weights[(size_t)n * E + e];
  } else {
    base = E * ff;
    count = shared;
    if (shared_w) scale = shared_w[n];
  }
  const T* row = y + (size_t)n * H;
  T* out = hs + (size_t)n * (top * ff + shared) + (size_t)k * ff;
#pragma unroll
  for (int r = 0; r < ER_ROWS / 4; ++r) {
    const int j = blockIdx.y * ER_ROWS + wave * (ER_ROWS / 4) + r;
    if (j >= count) break;
    const float a = unary_act(wave_dot(up + (size_t)(base + j) * H, row, H, vec, lane), act);
    if (lane == 0) out[j] = from_f32<T>(a * scale);
  }
}

// out[n, c] (+)= sum over the row's slots of down[c, slot's columns] . hs[n, slot's part]
template <typename T>
__global__ void __launch_bounds__(256)
expert_rows_down_kernel(const T* __restrict__ hs, const T* __restrict__ down, const int* __restrict__ chosen, int E, int top,
                        int ff, int shared, int H, bool vec, int accumulate, float* __restrict__ out) {
  const int n = blockIdx.x;
  const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
  const int total = E * ff + shared;
  const T* h = hs + (size_t)n * (top * ff + shared);
#pragma unroll
  for (int r = 0; r < ER_ROWS / 4; ++r) {
    const int c = blockIdx.y * ER_ROWS + wave * (ER_ROWS / 4) + r;
    if (c >= H) break;
    const T* w = down + (size_t)c * total;
    float acc = 0.f;
    for (int k = 0; k < top; ++k)
      acc += wave_dot(w + (size_t)chosen[(size_t)n * top + k] * ff, h + (size_t)k * ff, ff, vec, lane);
    if (shared) acc += wave_dot(w + (size_t)E * ff, h + (size_t)top * ff, shared, vec, lane);
    if (lane == 0) {
      float* o = out + (size_t)n * H + c;
      *o = accumulate ? *o + acc : acc;
    }
  }
}


// ---- gated experts ----------------------------------------------------------------------------------------
// An expert with a gate: down(act(g, u)) with g = W_gate t, u = W_up t and
//     act(g, u) = g' logistic(alpha g') (u' + shift) ,  g' = min(g, limit) ,  u' = clamp(u, -limit, limit).
// The stacked matrix holds, expert after expert, the rows [gate (ff) | up (ff)], and behind the last expert
// the shared one's [gate (shared) | up (shared)], which has a limit of its own.  The router's weight s
// multiplies the expert's INPUT t = s y (`on_input`: g and u are linear in t, so s multiplies both before
// the clamps) or its output (the activation times s).  An expert with weight 0 adds nothing either way.
struct GateTerms {
  float limit, limit_shared, alpha, shift;
  int on_input;
};

__device__ __forceinline__ float gated_value(float g, float u, float s, float limit, const GateTerms& k) {
  if (k.on_input) {
    g *= s;
    u *= s;
  }
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  const float a = g / (1.0f + expf(-k.alpha * g)) * (u + k.shift);
  return k.on_input ? a : a * s;
}

// out[n, j] for the E * ff + shared hidden channels j; gu float [n, 2 (E * ff + shared)] as the stacked matrix
// lays it; weights [n, E] (E == 0: none; a column of weight 1 for the shared part)
template <typename T>
__global__ void __launch_bounds__(256)
expert_gated_act_kernel(const float* __restrict__ gu, const float* __restrict__ weights, const float* __restrict__ shared_w,
                        int E, int ff, int shared, GateTerms k, T* __restrict__ out) {
  const int n = blockIdx.x;
  const int total = E * ff + shared;
  const float* row = gu + (size_t)n * 2 * total;
  for (int j = blockIdx.y * 256 + threadIdx.x; j < total; j += gridDim.y * 256) {
    float a;
    if (j < E * ff) {
      const int e = j / ff, c = j % ff;
      a = gated_value(row[2 * e * ff + c], row[2 * e * ff + ff + c], weights[(size_t)n * E + e], k.limit, k);
    } else {
      const int c = j - E * ff;
      a = gated_value(row[2 * E * ff + c], row[2 * E * ff + shared + c], 1.f, k.limit_shared, k);
      if (shared_w) a *= shared_w[n];
    }
    out[(size_t)n * total + j] = from_f32<T>(a);
  }
}

// the chosen experts alone: hs[n, k * ff + j] = act of expert chosen[n, k]'s rows j against y[n], and the shared
// expert's behind them; `up` is the stacked matrix [2 (E * ff + shared), H]
template <typename T>
__global__ void __launch_bounds__(256)
expert_rows_gated_up_kernel(const T* __restrict__ y, int H, const T* __restrict__ up, const int* __restrict__ chosen,
                            const float* __restrict__ weights, const float* __restrict__ shared_w, int E, int top, int ff,
                            int shared, GateTerms kt, bool vec, T* __restrict__ hs) {
  const int slots = top + (shared ? 1 : 0);
  const int n = blockIdx.x / slots, k = blockIdx.x % slots;
  const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
  int base, count;
  float scale = 1.f, limit = kt.limit_shared, after = 1.f;     // after: the shared expert's own weight, on its output
  if (k < top) {
    const int e = chosen[(size_t)n * top + k];
    base = 2 * e * ff;
    count = ff;
    scale = weights[(size_t)n * E + e];
    limit = kt.limit;
  } else {
    base = 2 * E * ff;
    count = shared;
    if (shared_w) after = shared_w[n];
  }
  const T* row = y + (size_t)n * H;
  T* out = hs + (size_t)n * (top * ff + shared) + (size_t)k * ff;
#pragma unroll
  for (int r = 0; r < ER_ROWS / 4; ++r) {
    const int j = blockIdx.y * ER_ROWS + wave * (ER_ROWS / 4) + r;
    if (j >= count) break;
    const float g = wave_dot(up + (size_t)(base + j) * H, row, H, vec, lane);
    const float u = wave_dot(up + (size_t)(base + count + j) * H, row, H, vec, lane);
    if (lane == 0) out[j] = from_f32<T>(gated_value(g, u, scale, limit, kt) * after);
  }
}

}  // namespace tl

using namespace tl;

extern "C" {

int tl_route(const void* h, int dt, int n, int W, const float* wr, int E, int groups, int keep, int top, int logistic,
             const float* correction, int two_largest, int normalise, float normalise_eps, float* shared_weight,
             const float* bias, float* weights, int* chosen, hipStream_t st) {
  TL_REQUIRE(n >= 0 && W > 0 && E > 0 && E <= RT_MAX_E && top > 0 && top <= E, "route: bad sizes n=%d W=%d E=%d top=%d (experts up to %d)",
             n, W, E, top, RT_MAX_E);
  TL_REQUIRE(groups >= 0 && (groups == 0 || (E % groups == 0 && keep > 0 && keep <= groups && keep * (E / groups) >= top)),
             "route: %d experts in %d groups of which %d are kept cannot give %d", E, groups, keep, top);
  TL_REQUIRE(h && wr && weights, "route: a buffer is missing");
  if (n == 0) return 0;
  const bool vec = W % 4 == 0 && (uintptr_t)h % 16 == 0 && (uintptr_t)wr % 16 == 0;
  TL_REQUIRE(dt == DT_F32 || dt == DT_BF16, "route: unknown dtype code %d", dt);
  const RouteTerms k{correction, two_largest, normalise, normalise_eps, shared_weight, bias};
  const bool few = n <= 64 && E > 4;             // fewer rows than compute units: more waves a row
  if (dt == DT_F32 && few)
    route_kernel<float, 1024><<<n, 1024, 0, st>>>((const float*)h, W, wr, E, groups, keep, top, logistic, k, weights, chosen, vec);
  else if (dt == DT_F32)
    route_kernel<float, 256><<<n, 256, 0, st>>>((const float*)h, W, wr, E, groups, keep, top, logistic, k, weights, chosen, vec);
  else if (few)
    route_kernel<bf16, 1024><<<n, 1024, 0, st>>>((const bf16*)h, W, wr, E, groups, keep, top, logistic, k, weights, chosen, vec);
  else
    route_kernel<bf16, 256><<<n, 256, 0, st>>>((const bf16*)h, W, wr, E, groups, keep, top, logistic, k, weights, chosen, vec);
  TL_LAUNCH_CHECK("route");
  return 0;
}

int tl_expert_act(const float* u, const float* weights, const float* shared_w, int n, int E, int ff, int total, int act_code,
                  float act_a, float act_b, void* out, int dt, hipStream_t st) {
  const UnaryAct act{act_code, act_a, act_b};
  TL_REQUIRE(n >= 0 && E >= 0 && ff > 0 && total >= E * ff && act_code >= 0 && act_code <= 2, "expert_act: bad sizes E=%d ff=%d total=%d act=%d",
             E, ff, total, act_code);
  TL_REQUIRE(u && out && (E == 0 || weights), "expert_act: a buffer is missing");
  if (n == 0) return 0;
  const dim3 grid(n, min((total + 255) / 256, 64));
  if (dt == DT_F32)
    expert_act_kernel<float><<<grid, 256, 0, st>>>(u, weights, shared_w, E, ff, total, act, (float*)out);
  else if (dt == DT_BF16)
    expert_act_kernel<bf16><<<grid, 256, 0, st>>>(u, weights, shared_w, E, ff, total, act, (bf16*)out);
  else
    TL_REQUIRE(false, "expert_act: unknown dtype code %d", dt);
  TL_LAUNCH_CHECK("expert_act");
  return 0;
}

// u (dtype udt) and out (dtype dt) of `total` elements, a multiple of 8, 16-byte aligned
int tl_unary_act(const void* u, int udt, long long total, int act_code, float act_a, float act_b, void* out, int dt, hipStream_t st) {
  const UnaryAct act{act_code, act_a, act_b};
  TL_REQUIRE(total >= 0 && total % 8 == 0 && act_code >= 0 && act_code <= 2, "unary_act: bad sizes total=%lld act=%d", total, act_code);
  TL_REQUIRE(u && out && (uintptr_t)u % 16 == 0 && (uintptr_t)out % 16 == 0, "unary_act: a buffer is missing or off 16 bytes");
  if (total == 0) return 0;
  const long long want = (total / 8 + 255) / 256;
  const unsigned blocks = (unsigned)(want < 8192 ? want : 8192);
  if (udt == DT_F32 && dt == DT_F32) unary_act_kernel<float, float><<<blocks, 256, 0, st>>>((const float*)u, (size_t)total, act, (float*)out);
  else if (udt == DT_F32 && dt == DT_BF16) unary_act_kernel<float, bf16><<<blocks, 256, 0, st>>>((const float*)u, (size_t)total, act, (bf16*)out);
  else if (udt == DT_BF16 && dt == DT_BF16) unary_act_kernel<bf16, bf16><<<blocks, 256, 0, st>>>((const bf16*)u, (size_t)total, act, (bf16*)out);
  else TL_REQUIRE(false, "unary_act: unknown dtype codes %d and %d", udt, dt);
  TL_LAUNCH_CHECK("unary_act");
  return 0;
}

// y [n, H], up [E * ff + shared, H], chosen int [n, top], weights [n, E] -> hs [n, top * ff + shared], all of dtype dt
int tl_expert_rows_up(const void* y, int H, const void* up, const int* chosen, const float* weights, const float* shared_w, int n, int E,
                      int top, int ff, int shared, int act_code, float act_a, float act_b, void* hs, int dt, hipStream_t st) {
  const UnaryAct act{act_code, act_a, act_b};
  TL_REQUIRE(n >= 0 && H > 0 && E > 0 && top > 0 && top <= E && ff > 0 && shared >= 0 && act_code >= 0 && act_code <= 2,
             "expert_rows_up: bad sizes H=%d E=%d top=%d ff=%d shared=%d act=%d", H, E, top, ff, shared, act_code);
  TL_REQUIRE(y && up && chosen && weights && hs, "expert_rows_up: a buffer is missing");
  TL_REQUIRE(dt == DT_F32 || dt == DT_BF16, "expert_rows_up: unknown dtype code %d", dt);
  if (n == 0) return 0;
  const int slots = top + (shared ? 1 : 0);
  const int most = ff > shared ? ff : shared;
  const dim3 grid(n * slots, (most + ER_ROWS - 1) / ER_ROWS);
  const int per = dt == DT_BF16 ? 8 : 4;
  const bool vec = H % per == 0 && (uintptr_t)y % 16 == 0 && (uintptr_t)up % 16 == 0;
  if (dt == DT_F32)
    expert_rows_up_kernel<float><<<grid, 256, 0, st>>>((const float*)y, H, (const float*)up, chosen, weights, shared_w, E, top, ff, shared, act, vec,
                                                       (float*)hs);
  else
    expert_rows_up_kernel<bf16><<<grid, 256, 0, st>>>((const bf16*)y, H, (const bf16*)up, chosen, weights, shared_w, E, top, ff, shared, act, vec,
                                                      (bf16*)hs);
  TL_LAUNCH_CHECK("expert_rows_up");
  return 0;
}

// hs [n, top * ff + shared], down [H, E * ff + shared] of dtype dt -> out float [n, H], added to or stored
int tl_expert_rows_down(const void* hs, const void* down, const int* chosen, int n, int E, int top, int ff, int shared, int H,
                        int accumulate, float* out, int dt, hipStream_t st) {
  TL_REQUIRE(n >= 0 && H > 0 && E > 0 && top > 0 && top <= E && ff > 0 && shared >= 0, "expert_rows_down: bad sizes H=%d E=%d top=%d ff=%d shared=%d",
             H, E, top, ff, shared);
  TL_REQUIRE(hs && down && chosen && out, "expert_rows_down: a buffer is missing");
  TL_REQUIRE(dt == DT_F32 || dt == DT_BF16, "expert_rows_down: unknown dtype code %d", dt);
  if (n == 0) return 0;
  const dim3 grid(n, (H + ER_ROWS - 1) / ER_ROWS);
  const int per = dt == DT_BF16 ? 8 : 4;
  const bool vec = ff % per == 0 && shared % per == 0 && (uintptr_t)hs % 16 == 0 && (uintptr_t)down % 16 == 0;
  if (dt == DT_F32)
    expert_rows_down_kernel<float><<<grid, 256, 0, st>>>((const float*)hs, (const float*)down, chosen, E, top, ff, shared, H, vec, accumulate, out);
  else
    expert_rows_down_kernel<bf16><<<grid, 256, 0, st>>>((const bf16*)hs, (const bf16*)down, chosen, E, top, ff, shared, H, vec, accumulate, out);
  TL_LAUNCH_CHECK("expert_rows_down");
  return 0;
}

// gu float [n, 2 (E * ff + shared)], weights float [n, E] (E == 0: none) -> out [n, E * ff + shared] of dtype dt
int tl_expert_gated_act(const float* gu, const float* weights, const float* shared_w, int n, int E, int ff, int shared, float limit, float limit_shared,
                        float alpha, float shift, int on_input, void* out, int dt, hipStream_t st) {
  TL_REQUIRE(n >= 0 && E >= 0 && ff >= 0 && shared >= 0 && E * ff + shared > 0, "expert_gated_act: bad sizes E=%d ff=%d shared=%d", E, ff, shared);
  TL_REQUIRE(gu && out && (E == 0 || weights), "expert_gated_act: a buffer is missing");
  TL_REQUIRE(dt == DT_F32 || dt == DT_BF16, "expert_gated_act: unknown dtype code %d", dt);
  if (n == 0) return 0;
  const int total = E * ff + shared;
  const dim3 grid(n, min((total + 255) / 256, 64));
  const GateTerms k{limit, limit_shared, alpha, shift, on_input};
  if (dt == DT_F32) expert_gated_act_kernel<float><<<grid, 256, 0, st>>>(gu, weights, shared_w, E, ff, shared, k, (float*)out);
  else expert_gated_act_kernel<bf16><<<grid, 256, 0, st>>>(gu, weights, shared_w, E, ff, shared, k, (bf16*)out);
  TL_LAUNCH_CHECK("expert_gated_act");
  return 0;
}

// y [n, H], up [2 (E * ff + shared), H], chosen int [n, top], weights [n, E] -> hs [n, top * ff + shared], all of dtype dt
int tl_expert_rows_gated_up(const void* y, int H, const void* up, const int* chosen, const float* weights, const float* shared_w, int n,
                            int E, int top, int ff, int shared, float limit, float limit_shared, float alpha, float shift, int on_input, void* hs,
                            int dt, hipStream_t st) {
  TL_REQUIRE(n >= 0 && H > 0 && E > 0 && top > 0 && top <= E && ff > 0 && shared >= 0,
             "expert_rows_gated_up: bad sizes H=%d E=%d top=%d ff=%d shared=%d", H, E, top, ff, shared);
  TL_REQUIRE(y && up && chosen && weights && hs, "expert_rows_gated_up: a buffer is missing");
  TL_REQUIRE(dt == DT_F32 || dt == DT_BF16, "expert_rows_gated_up: unknown dtype code %d", dt);
  if (n == 0) return 0;
  const int slots = top + (shared ? 1 : 0);
  const int most = ff > shared ? ff : shared;
  const dim3 grid(n * slots, (most + ER_ROWS - 1) / ER_ROWS);
  const int per = dt == DT_BF16 ? 8 : 4;
  const bool vec = H % per == 0 && (uintptr_t)y % 16 == 0 && (uintptr_t)up % 16 == 0;
  const GateTerms k{limit, limit_shared, alpha, shift, on_input};
  if (dt == DT_F32)
    expert_rows_gated_up_kernel<float><<<grid, 256, 0, st>>>((const float*)y, H, (const float*)up, chosen, weights, shared_w, E, top, ff, shared, k,
                                                             vec, (float*)hs);
  else
    expert_rows_gated_up_kernel<bf16><<<grid, 256, 0, st>>>((const bf16*)y, H, (const bf16*)up, chosen, weights, shared_w, E, top, ff, shared, k,
                                                            vec, (bf16*)hs);
  TL_LAUNCH_CHECK("expert_rows_gated_up");
  return 0;
}

}  // extern "C"
