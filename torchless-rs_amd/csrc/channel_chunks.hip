// Linear attention with a decay per key channel, plain or by the delta rule, by chunks of rows on the
// matrix cores: bfloat16 steps that bring many rows (see channel_linear.hip for the mechanism).  A
// sequence's new rows are cut into chunks of CC = 64 counted from the step's first row; with i, j the places in a
// chunk, S the state before it and D_i the product of the decays of rows 0 .. i (a factor per channel),
//
//   A_ij = sum_d k_i k_j D_i/D_j (j < i) ,   B_ij = sum_d q_i k_j D_i/D_j (j <= i)
//   (I + diag(beta) A) [W | V'] = diag(beta) [D k | V]           (plain: V' = V, no W)
//   U = V' - W S ,   o = (D q) S + B U ,   S <- D_last S + (D_last/D k)^T U
//
// (the delta rule written for a chunk at once, as in Yang et al., Parallelizing Linear Transformers with
// the Delta Rule over Sequence Length).  Two kernels:
//
//   local  one workgroup a chunk and head: convolution, unit norms and decays of its rows, A and B, the solution of
//          the triangular system by blocks of 16 rows, and every operand of the second kernel in the order in which a
//          wave's lanes take it
//   carry  one wave 16 columns of a head's state, through the chunks of a sequence in their order, with the state in
//          its registers in float: a product's result is the next one's operand without leaving them
//
// Decays are kept as logarithms (base 2) summed inside blocks of 16 rows, with the blocks' sums beside them: every
// factor D_i/D_j with j <= i is then 2 to a sum of numbers that are none above 0, whatever the decays; inside a block
// of 16 rows A and B are summed in float without the matrix cores.  A float that becomes an operand goes in two
// bfloat16 terms, x = hi + lo (16 bits of its mantissa), and products of two such in three products; only the operands
// that nothing but a row's own result depends on (D q and B) are rounded to one.  Sums are float.
#include "channel_linear.hpp"
#include "chunks.hpp"

namespace tl {

constexpr int CC = 64;               // rows of a chunk
constexpr int CC_MAX_DK = 128;
constexpr int FRAG = 512;            // elements of an operand of 16 x 32, lane by lane
constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ f32x4 mfma16(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ void split8(const float* x, bf16x8& hi, bf16x8& lo) {
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    hi[e] = (bf16)x[e];
    lo[e] = (bf16)(x[e] - (float)hi[e]);
  }
}
// two results of 16 rows each (a lane holds rows 4g .. 4g+3 of one column) as the operand of a product over those 32 rows
__device__ __forceinline__ void split_tiles(const f32x4& a, const f32x4& b, bf16x8& hi, bf16x8& lo) {
  const float x[8] = {a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
  split8(x, hi, lo);
}
__device__ __forceinline__ f32x4 ld4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ float ex2(float x) { return __builtin_amdgcn_exp2f(x); }

// operands that `local` leaves for a chunk and head, in FRAGs: W hi, W lo (delta rule only) [4][DK/32]; (D_last/D k)^T hi, lo
// [DK/16][2]; D q [4][DK/32]; B [4][2]
template <int DK, bool DELTA> struct Record {
  static constexpr int KS = DK / 32;                     // steps over the channels
  static constexpr int W_HI = 0, W_LO = DELTA ? 4 * KS : 0;
  static constexpr int K_HI = DELTA ? 8 * KS : 0, K_LO = K_HI + DK / 8, Q = K_LO + DK / 8, B = Q + 4 * KS;
  static constexpr int FRAGS = B + 8;
};

struct ChunkArgs {
  const float* proj;
  int width, v_off;
  const float* z;                  // [n, H * dk]: the decays' second step without its bias
  const float* conv_state;
  long long stride;
  const int* cu;
  const int* slots;
  int B;
};

// 16 rows n0 .. of one channel (column c of proj), through the convolution if there is one; rows behind `rows` are zeros
template <int ROWS>
__device__ __forceinline__ void channel_run(const ChunkArgs& a, const ChannelTerms& t, int C, int n0, int seq_i0, int rows, const float* st, int c,
                                            float* out) {
  float cur[ROWS];
  const float* p = a.proj + (size_t)n0 * a.width + c;
#pragma unroll
  for (int r = 0; r < ROWS; ++r) cur[r] = r < rows ? p[(size_t)r * a.width] : 0.f;
  if (!t.taps) {
#pragma unroll
    for (int r = 0; r < ROWS; ++r) out[r] = cur[r];
    return;
  }
  float w[CL_MAX_TAPS], win[CL_MAX_TAPS];              // right-aligned: the last is the present row's
#pragma unroll
  for (int j = 0; j < CL_MAX_TAPS; ++j) {
    const int back = CL_MAX_TAPS - 1 - j;
    w[j] = back < t.taps ? t.conv_w[(size_t)c * t.taps + t.taps - 1 - back] : 0.f;
    win[j] = 0.f;
    if (back > 0 && back < t.taps) {
      const int src = seq_i0 - back;
      win[j] = src >= 0 ? p[-(ptrdiff_t)back * a.width] : st[(size_t)(t.taps - 1 + src) * C + c];
    }
  }
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    win[CL_MAX_TAPS - 1] = cur[r];
    float acc = 0.f;
#pragma unroll
    for (int j = 0; j < CL_MAX_TAPS; ++j) acc = fmaf(w[j], win[j], acc);
    out[r] = r < rows ? cl_silu(acc) : 0.f;
#pragma unroll
    for (int j = 0; j + 1 < CL_MAX_TAPS; ++j) win[j] = win[j + 1];
  }
}

template <int DK> constexpr size_t local_lds() {
  return sizeof(float) * (3 * CC * (DK + 4) + 2 * CC * (CC + 4) + 4 * DK + CC + 4 * 16 * 20);
}

// grid (chunks, H), 4 * DK threads
template <int DK, bool DELTA>
__global__ void __launch_bounds__(4 * DK)
channel_local_kernel(ChunkArgs a, ChannelTerms t, bf16* __restrict__ rec, float* __restrict__ gam, float* __restrict__ uf, int nct) {
  using R = Record<DK, DELTA>;
  constexpr int LD = DK + 4, MLD = CC + 4, KS = DK / 32, NW = DK / 16, NT = 4 * DK;
  extern __shared__ __attribute__((aligned(16))) float cc_lds[];
  float* qs = cc_lds;                    // [CC][LD]
  float* ks = qs + CC * LD;              // [CC][LD]
  float* ls = ks + CC * LD;              // [CC][LD]: log2 of the decays, summed from the block's first row to this one
  float* Ms = ls + CC * LD;              // [CC][MLD]: diag(beta) A
  float* Bs = Ms + CC * MLD;             // [CC][MLD]
  float* tot = Bs + CC * MLD;            // [4][DK]: a block's sum
  float* bt = tot + 4 * DK;              // [CC]
  float* Ti = bt + CC;                   // [4][16][20]: inverses of the blocks on the diagonal
  Chunk ch;
  const int c = blockIdx.x, h = blockIdx.y;
  if (!find_chunk(c, a.cu, a.B, CC, ch)) return;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE, m = lane % 16, g = lane / 16;
  const int kh = h / (t.H / t.G), Q = t.G * t.dk, C = 2 * Q + t.H * t.dv;
  const int seq0 = ch.row0 - a.cu[ch.b];             // the chunk's first row counted from the step's first of the sequence
  const float* st = t.taps ? a.conv_state + (long long)a.slots[ch.b] * a.stride : nullptr;
  {
    const int d = tid % DK, i0 = (tid / DK) * 16;
    float x[16];
    const bool in = d < t.dk;
    const int rows = in ? ch.rows - i0 : 0, n0 = ch.row0 + i0;
    if (rows > 0) channel_run<16>(a, t, C, n0, seq0 + i0, rows, st, kh * t.dk + d, x);
#pragma unroll
    for (int r = 0; r < 16; ++r) qs[(i0 + r) * LD + d] = rows > 0 ? x[r] : 0.f;
    if (rows > 0) channel_run<16>(a, t, C, n0, seq0 + i0, rows, st, Q + kh * t.dk + d, x);
#pragma unroll
    for (int r = 0; r < 16; ++r) ks[(i0 + r) * LD + d] = rows > 0 ? x[r] : 0.f;
    const float rate = t.rate ? -expf(t.rate[h]) : 0.f;
    const float bias = in && t.bias ? t.bias[h * t.dk + d] : 0.f;
    const float* zp = a.z + (size_t)n0 * t.H * t.dk + h * t.dk + d;
#pragma unroll
    for (int r = 0; r < 16; ++r) x[r] = r < rows ? zp[(size_t)r * t.H * t.dk] : 0.f;
    float sum = 0.f;
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      if (r < rows) sum += cl_log_decay(x[r] + bias, t.rate != nullptr, rate, t.inv_tau) * LOG2E;
      ls[(i0 + r) * LD + d] = sum;
    }
    tot[(tid / DK) * DK + d] = sum;
    if (DELTA && tid < CC)
      bt[tid] = tid < ch.rows ? cl_sigmoid(a.proj[(size_t)(ch.row0 + tid) * a.width + t.b_off + h]) : 0.f;
  }
  __syncthreads();
  {                                                    // q and k of every row: unit vectors, the factor on q
    constexpr int P = NT / CC, E = DK / P;             // lanes a row, channels a lane
    const int i = tid / P, e0 = (tid % P) * E;
    f32x4 xq[E / 4], xk[E / 4];
    float sq = 0.f, sk = 0.f;
#pragma unroll
    for (int e = 0; e < E / 4; ++e) {
      xq[e] = ld4(qs + i * LD + e0 + 4 * e);
      xk[e] = ld4(ks + i * LD + e0 + 4 * e);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        sq += xq[e][j] * xq[e][j];
        sk += xk[e][j] * xk[e][j];
      }
    }
    float fq = t.qscale, fk = 1.f;
    if (t.unit_eps >= 0.f) {
#pragma unroll
      for (int o = 1; o < P; o *= 2) {
        sq += __shfl_xor(sq, o, WAVE);
        sk += __shfl_xor(sk, o, WAVE);
      }
      fq *= 1.0f / sqrtf(sq + t.unit_eps);
      fk = 1.0f / sqrtf(sk + t.unit_eps);
    }
#pragma unroll
    for (int e = 0; e < E / 4; ++e) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        xq[e][j] *= fq;
        xk[e][j] *= fk;
      }
      *reinterpret_cast<f32x4*>(qs + i * LD + e0 + 4 * e) = xq[e];
      *reinterpret_cast<f32x4*>(ks + i * LD + e0 + 4 * e) = xk[e];
    }
  }
  __syncthreads();

  // A (role 0) and B (role 1): blocks on the diagonal in float, those below it on the matrix cores
  for (int task = (DELTA ? 0 : 4) + wave; task < 8; task += NW) {
    const int role = task / 4, w4 = task % 4;
    const float* rs = role ? qs : ks;
    float* out = role ? Bs : Ms;
    {
      const int i = 16 * w4 + m, j0 = 16 * w4 + 4 * g;
      float acc[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
      for (int d = 0; d < DK; d += 4) {
        const f32x4 x = ld4(rs + i * LD + d), li = ld4(ls + i * LD + d);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const f32x4 y = ld4(ks + (j0 + j) * LD + d), lj = ld4(ls + (j0 + j) * LD + d);
#pragma unroll
          for (int e = 0; e < 4; ++e) acc[j] = fmaf(x[e] * y[e], ex2(li[e] - lj[e]), acc[j]);
        }
      }
      const float f = role ? 1.f : bt[i];
      f32x4 r;
#pragma unroll
      for (int j = 0; j < 4; ++j) r[j] = j0 + j < i + role ? acc[j] * f : 0.f;      // (nothing of what lies above is read)
      *reinterpret_cast<f32x4*>(out + i * MLD + j0) = r;
    }
    for (int pair = 0; pair < 2; ++pair) {
      // wave 0: (3, 0); 1: (3, 1); 2: (3, 2), (1, 0); 3: (2, 0), (2, 1)
      if (pair == 1 && w4 < 2) break;
      const int I = w4 == 3 ? 2 : (w4 == 2 && pair ? 1 : 3), J = w4 == 3 ? pair : (w4 == 2 && pair ? 0 : w4);
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const int d = 32 * s + 8 * g;
        float x[8], y[8];
#pragma unroll
        for (int q4 = 0; q4 < 2; ++q4) {
          const f32x4 xr = ld4(rs + (16 * I + m) * LD + d + 4 * q4), li = ld4(ls + (16 * I + m) * LD + d + 4 * q4);
          const f32x4 yr = ld4(ks + (16 * J + m) * LD + d + 4 * q4), lj = ld4(ls + (16 * J + m) * LD + d + 4 * q4);
          f32x4 between = ld4(tot + J * DK + d + 4 * q4) - lj;
          for (int M = J + 1; M < I; ++M) between += ld4(tot + M * DK + d + 4 * q4);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            x[4 * q4 + e] = xr[e] * ex2(li[e]);
            y[4 * q4 + e] = yr[e] * ex2(between[e]);
          }
        }
        bf16x8 xh, xl, yh, yl;
        split8(x, xh, xl);
        split8(y, yh, yl);
        acc = mfma16(xh, yh, acc);
        acc = mfma16(xh, yl, acc);
        acc = mfma16(xl, yh, acc);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * I + 4 * g + r;
        out[i * MLD + 16 * J + m] = acc[r] * (role ? 1.f : bt[i]);
      }
    }
  }
  __syncthreads();

  if (DELTA && wave < 4 && lane < 16) {                // column `lane` of the inverse of a block on the diagonal
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float s0 = i == lane ? 1.f : 0.f, s1 = 0.f;
      const float* Mr = Ms + (16 * wave + i) * MLD + 16 * wave;
#pragma unroll
      for (int j = 0; j < i; ++j) {
        if (j % 2) s1 = fmaf(-Mr[j], x[j], s1);
        else s0 = fmaf(-Mr[j], x[j], s0);
      }
      x[i] = s0 + s1;
      Ti[(wave * 16 + i) * 20 + lane] = x[i];
    }
  }
  bf16* mine = rec + ((size_t)c * t.H + h) * R::FRAGS * FRAG;
  // operands: lane (m, g) of a FRAG holds row m and the eight columns 4g .. 4g+3, 16 + 4g .. 16 + 4g+3 of its 32
  for (int f = wave; f < 4 * KS; f += NW) {            // D q
    const int mt = f / KS, s = f % KS, i = 16 * mt + m;
    bf16x8 v;
#pragma unroll
    for (int q4 = 0; q4 < 2; ++q4) {
      const int d = 32 * s + 16 * q4 + 4 * g;
      const f32x4 x = ld4(qs + i * LD + d);
      f32x4 l = ld4(ls + i * LD + d);
      for (int M = 0; M < mt; ++M) l += ld4(tot + M * DK + d);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[4 * q4 + e] = (bf16)(x[e] * ex2(l[e]));
    }
    *reinterpret_cast<bf16x8*>(mine + (size_t)(R::Q + f) * FRAG + lane * 8) = v;
  }
  for (int f = wave; f < DK / 8; f += NW) {            // (D_last / D k)^T
    const int d = 16 * (f / 2) + m, s = f % 2;
    float x[8];
#pragma unroll
    for (int q4 = 0; q4 < 2; ++q4) {
      const int J = 2 * s + q4;
      float rest = 0.f;
      for (int M = J; M < 4; ++M) rest += tot[M * DK + d];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int j = 16 * J + 4 * g + e;
        x[4 * q4 + e] = ks[j * LD + d] * ex2(rest - ls[j * LD + d]);
      }
    }
    bf16x8 hi, lo;
    split8(x, hi, lo);
    *reinterpret_cast<bf16x8*>(mine + (size_t)(R::K_HI + f) * FRAG + lane * 8) = hi;
    *reinterpret_cast<bf16x8*>(mine + (size_t)(R::K_LO + f) * FRAG + lane * 8) = lo;
  }
  for (int f = wave; f < 8; f += NW) {                 // B
    const int mt = f / 2, s = f % 2, i = 16 * mt + m;
    bf16x8 v;
#pragma unroll
    for (int q4 = 0; q4 < 2; ++q4) {
      const int J = 2 * s + q4;
      f32x4 x = {0.f, 0.f, 0.f, 0.f};
      if (J <= mt) x = ld4(Bs + i * MLD + 16 * J + 4 * g);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[4 * q4 + e] = (bf16)x[e];
    }
    *reinterpret_cast<bf16x8*>(mine + (size_t)(R::B + f) * FRAG + lane * 8) = v;
  }
  if (tid < DK) gam[((size_t)c * t.H + h) * DK + tid] = ex2(tot[tid] + tot[DK + tid] + tot[2 * DK + tid] + tot[3 * DK + tid]);
  __syncthreads();                                     // q has been read: its place takes W

  bf16* w_hi = reinterpret_cast<bf16*>(qs);            // [CC][LD]
  bf16* w_lo = w_hi + CC * LD;
  for (int ct = (DELTA ? 0 : DK / 16) + wave; ct < DK / 16 + nct; ct += NW) {
    const bool is_w = ct < DK / 16;
    f32x4 x[4];                                        // rows 16 I + 4 g .. of column m
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      if (is_w) {
        const int d = 16 * ct + m;
        float before = 0.f;
        for (int M = 0; M < I; ++M) before += tot[M * DK + d];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = 16 * I + 4 * g + r;
          x[I][r] = bt[i] * ks[i * LD + d] * ex2(before + ls[i * LD + d]);
        }
      } else {
        const int col = 16 * (ct - DK / 16) + m, i0 = 16 * I + 4 * g;
        float v[4] = {0.f, 0.f, 0.f, 0.f};
        if (col < t.dv && i0 < ch.rows) channel_run<4>(a, t, C, ch.row0 + i0, seq0 + i0, ch.rows - i0, st, a.v_off + h * t.dv + col, v);
#pragma unroll
        for (int r = 0; r < 4; ++r) x[I][r] = DELTA ? bt[i0 + r] * v[r] : v[r];
      }
    }
    if constexpr (DELTA) {
      bf16x8 ph[2], pl[2];                             // solved blocks 0, 1 and 2, 3 as operands
#pragma unroll
      for (int I = 0; I < 4; ++I) {
        f32x4 acc = x[I];
#pragma unroll
        for (int p = 0; p < 2; ++p) {
          if (2 * p >= I) continue;
          float mm[8];
          const f32x4 m0 = ld4(Ms + (16 * I + m) * MLD + 32 * p + 4 * g);
          f32x4 m1 = {0.f, 0.f, 0.f, 0.f};
          if (2 * p + 1 < I) m1 = ld4(Ms + (16 * I + m) * MLD + 32 * p + 16 + 4 * g);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            mm[e] = -m0[e];
            mm[4 + e] = -m1[e];
          }
          bf16x8 mh, ml;
          split8(mm, mh, ml);
          acc = mfma16(mh, ph[p], acc);
          acc = mfma16(mh, pl[p], acc);
          acc = mfma16(ml, ph[p], acc);
        }
        const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
        bf16x8 th, tl, rh, rl;
        split_tiles(ld4(Ti + (I * 16 + m) * 20 + 4 * g), zero, th, tl);
        split_tiles(acc, zero, rh, rl);
        f32x4 y = mfma16(th, rh, zero);
        y = mfma16(th, rl, y);
        y = mfma16(tl, rh, y);
        x[I] = y;
        if (I == 0) split_tiles(x[0], zero, ph[0], pl[0]);
        if (I == 1) split_tiles(x[0], x[1], ph[0], pl[0]);
        if (I == 2) split_tiles(x[2], zero, ph[1], pl[1]);
      }
    }
    if (is_w) {
#pragma unroll
      for (int I = 0; I < 4; ++I)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int at = (16 * I + 4 * g + r) * LD + 16 * ct + m;
          const float v = -x[I][r];
          const bf16 hi = (bf16)v;
          w_hi[at] = hi;
          w_lo[at] = (bf16)(v - (float)hi);
        }
    } else {
      float* up = uf + (((size_t)c * t.H + h) * nct + ct - DK / 16) * (CC * 16);
#pragma unroll
      for (int I = 0; I < 4; ++I) *reinterpret_cast<f32x4*>(up + (I * WAVE + lane) * 4) = x[I];
    }
  }
  if constexpr (DELTA) {
    __syncthreads();
    for (int f = wave; f < 8 * KS; f += NW) {          // -W, hi and lo
      const int part = f / (4 * KS), mt = (f % (4 * KS)) / KS, s = f % KS;
      const bf16* src = (part ? w_lo : w_hi) + (16 * mt + m) * LD + 32 * s + 4 * g;
      const bf16x4 p0 = *reinterpret_cast<const bf16x4*>(src), p1 = *reinterpret_cast<const bf16x4*>(src + 16);
      bf16x8 v;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        v[e] = p0[e];
        v[4 + e] = p1[e];
      }
      *reinterpret_cast<bf16x8*>(mine + (size_t)((part ? R::W_LO : R::W_HI) + f % (4 * KS)) * FRAG + lane * 8) = v;
    }
  }
}

template <int DK, bool DELTA> constexpr size_t carry_lds() { return (size_t)Record<DK, DELTA>::FRAGS * FRAG * sizeof(bf16) + DK * sizeof(float); }

// grid (H, parts of 64 columns, B), 4 waves
template <int DK, bool DELTA>
__global__ void __launch_bounds__(256, 1)
channel_carry_kernel(const bf16* __restrict__ rec, const float* __restrict__ gam, const float* __restrict__ uf, int nct, int H, int dk, int dv,
                     float* __restrict__ state, long long stride, const int* __restrict__ cu, const int* __restrict__ slots,
                     float* __restrict__ o) {
  using R = Record<DK, DELTA>;
  constexpr int KS = DK / 32, MT = DK / 16, LOADS = R::FRAGS * FRAG * 2 / (256 * 16);
  extern __shared__ __attribute__((aligned(16))) bf16 cy_lds[];
  float* gs = reinterpret_cast<float*>(cy_lds + R::FRAGS * FRAG);       // [DK]
  const int h = blockIdx.x, b = blockIdx.z;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE, m = lane % 16, g = lane / 16;
  const int ct = blockIdx.y * 4 + wave, col = 16 * ct + m;
  int first = 0;
  for (int s = 0; s < b; ++s) first += (cu[s + 1] - cu[s] + CC - 1) / CC;
  const int row0 = cu[b], n = cu[b + 1] - row0, chunks = (n + CC - 1) / CC;
  if (chunks == 0) return;
  const bool active = ct < nct;
  const bool ok = active && col < dv;
  float* S_g = state + (long long)slots[b] * stride + ((size_t)h * dv + (ok ? col : 0)) * dk;
  f32x4 S[MT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * mt + 4 * g + r;
      S[mt][r] = ok && d < dk ? S_g[d] : 0.f;
    }
  f32x4 stage[LOADS], gst, u0[4], un[4];
  auto load = [&](int c) {
    const size_t at = (size_t)(first + c) * H + h;
    const f32x4* src = reinterpret_cast<const f32x4*>(rec + at * R::FRAGS * FRAG);
#pragma unroll
    for (int e = 0; e < LOADS; ++e) stage[e] = src[e * 256 + tid];
    if (tid < DK / 4) gst = ld4(gam + at * DK + 4 * tid);
    if (active) {
      const float* up = uf + (at * nct + ct) * (CC * 16);
#pragma unroll
      for (int I = 0; I < 4; ++I) un[I] = ld4(up + (I * WAVE + lane) * 4);
    }
  };
  auto frag = [&](int f) { return *reinterpret_cast<const bf16x8*>(cy_lds + f * FRAG + lane * 8); };
  load(0);
  for (int c = 0; c < chunks; ++c) {
    __syncthreads();                                   // the chunk before has been worked on
#pragma unroll
    for (int e = 0; e < LOADS; ++e) reinterpret_cast<f32x4*>(cy_lds)[e * 256 + tid] = stage[e];
    if (tid < DK / 4) *reinterpret_cast<f32x4*>(gs + 4 * tid) = gst;
#pragma unroll
    for (int I = 0; I < 4; ++I) u0[I] = un[I];
    __syncthreads();
    if (c + 1 < chunks) load(c + 1);
    if (!active) continue;
    f32x4 out[4];
#pragma unroll
    for (int I = 0; I < 4; ++I) out[I] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      bf16x8 sh, sl;
      split_tiles(S[2 * s], S[2 * s + 1], sh, sl);
#pragma unroll
      for (int I = 0; I < 4; ++I) {
        if constexpr (DELTA) {
          const bf16x8 wh = frag(R::W_HI + I * KS + s), wl = frag(R::W_LO + I * KS + s);
          u0[I] = mfma16(wh, sh, u0[I]);
          u0[I] = mfma16(wh, sl, u0[I]);
          u0[I] = mfma16(wl, sh, u0[I]);
        }
        const bf16x8 qf = frag(R::Q + I * KS + s);
        out[I] = mfma16(qf, sh, out[I]);
        out[I] = mfma16(qf, sl, out[I]);
      }
    }
    bf16x8 uh[2], ul[2];
    split_tiles(u0[0], u0[1], uh[0], ul[0]);
    split_tiles(u0[2], u0[3], uh[1], ul[1]);
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      S[mt] *= ld4(gs + 16 * mt + 4 * g);
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        const bf16x8 kh = frag(R::K_HI + 2 * mt + s), kl = frag(R::K_LO + 2 * mt + s);
        S[mt] = mfma16(kh, uh[s], S[mt]);
        S[mt] = mfma16(kh, ul[s], S[mt]);
        S[mt] = mfma16(kl, uh[s], S[mt]);
      }
    }
#pragma unroll
    for (int I = 0; I < 4; ++I) {
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        if (2 * s > I) continue;                       // (B is zero above the diagonal)
        const bf16x8 bf = frag(R::B + 2 * I + s);
        out[I] = mfma16(bf, uh[s], out[I]);
        out[I] = mfma16(bf, ul[s], out[I]);
      }
      if (ok) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = c * CC + 16 * I + 4 * g + r;
          if (i < n) o[((size_t)(row0 + i) * H + h) * dv + col] = out[I][r];
        }
      }
    }
  }
  if (!ok) return;
#pragma unroll
  for (int mt = 0; mt < MT; ++mt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * mt + 4 * g + r;
      if (d < dk) S_g[d] = S[mt][r];
    }
}

template <int DK, bool DELTA>
static int launch_chunks(const ChunkArgs& a, const ChannelTerms& t, int chunks, bf16* rec, float* gam, float* uf, float* state, long long stride,
                         float* o, hipStream_t st) {
  static bool raised = false;
  if (!raised) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&channel_local_kernel<DK, DELTA>),
                                       hipFuncAttributeMaxDynamicSharedMemorySize, (int)local_lds<DK>());
    if (e == hipSuccess)
      e = hipFuncSetAttribute(reinterpret_cast<const void*>(&channel_carry_kernel<DK, DELTA>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, (int)carry_lds<DK, DELTA>());
    if (e != hipSuccess) {
      set_error("channel_chunks: cannot have %zu and %zu bytes of LDS: %s", local_lds<DK>(), carry_lds<DK, DELTA>(), hipGetErrorString(e));
      return 2;
    }
    raised = true;
  }
  const int nct = (t.dv + 15) / 16;
  channel_local_kernel<DK, DELTA><<<dim3(chunks, t.H), 4 * DK, local_lds<DK>(), st>>>(a, t, rec, gam, uf, nct);
  TL_LAUNCH_CHECK("channel_local");
  channel_carry_kernel<DK, DELTA><<<dim3(t.H, (nct + 3) / 4, a.B), 256, carry_lds<DK, DELTA>(), st>>>(rec, gam, uf, nct, t.H, t.dk, t.dv, state,
                                                                                                 stride, a.cu, a.slots, o);
  TL_LAUNCH_CHECK("channel_carry");
  return 0;
}

// hi and lo of `cols` columns of x side by side, each padded with zeros to `pad` columns: out[n, j] and out[n, pad + j]
__global__ void __launch_bounds__(256)
split_columns_kernel(const float* __restrict__ x, int stride, int cols, int pad, int total, bf16* __restrict__ out) {
  const int e = blockIdx.x * 256 + threadIdx.x;
  if (e >= total) return;
  const int n = e / pad, j = e % pad;
  const float v = j < cols ? x[(size_t)n * stride + j] : 0.f;
  const bf16 hi = (bf16)v;
  out[(size_t)n * 2 * pad + j] = hi;
  out[(size_t)n * 2 * pad + pad + j] = (bf16)(v - (float)hi);
}

}  // namespace tl

using namespace tl;

extern "C" {

int tl_channel_chunk(void) { return CC; }

// FRAGs of a chunk and head, in bfloat16 elements, and the padded size of a key head
int tl_channel_record(int dk, int delta) {
  if (dk <= 64) return (delta ? Record<64, true>::FRAGS : Record<64, false>::FRAGS) * FRAG;
  return (delta ? Record<128, true>::FRAGS : Record<128, false>::FRAGS) * FRAG;
}
int tl_channel_padded(int dk) { return dk <= 64 ? 64 : 128; }

int tl_split_columns(const float* x, int stride, int cols, int pad, int n, void* out, hipStream_t st) {
  TL_REQUIRE(n >= 0 && cols > 0 && cols <= pad && stride >= cols && x && out, "split_columns: bad arguments n=%d cols=%d pad=%d", n, cols, pad);
  TL_REQUIRE((long long)n * pad < 2147483647LL - 256, "split_columns: too many rows");
  if (n == 0) return 0;
  const int total = n * pad;
  split_columns_kernel<<<(total + 255) / 256, 256, 0, st>>>(x, stride, cols, pad, total, (bf16*)out);
  TL_LAUNCH_CHECK("split_columns");
  return 0;
}

// proj [n, width] float = [q | k | v | ..]; z [n, H*dk] float (second step of the decays, without the bias); `chunks`: the step's
// chunks.  Scratch: rec chunks*H*tl_channel_record, gam chunks*H*tl_channel_padded floats, uf chunks*H*ceil(dv/16)*1024 floats.
// o float [n, H*dv].
int tl_channel_chunks(const float* proj, int width, int G, int H, int dk, int dv, int b_off, int taps, const float* conv_w, const float* bias,
                      const float* rate, float inv_tau, float qscale, float unit_eps, const float* z, const float* conv_state,
                      long long conv_stride, float* state, long long stride, const int* cu, const int* slots, int n, int B, int chunks,
                      void* rec, float* gam, float* uf, float* o, hipStream_t st) {
  TL_REQUIRE(n > 0 && B > 0 && B <= 65535 && G > 0 && H > 0 && H <= 65535 && H % G == 0 && chunks > 0, "channel_chunks: bad sizes n=%d B=%d G=%d H=%d chunks=%d",
             n, B, G, H, chunks);
  TL_REQUIRE(dk > 0 && dk <= CC_MAX_DK && dv > 0 && dv <= CL_MAX_D, "channel_chunks: heads of %d and %d are not served (up to %d and %d)", dk, dv,
             CC_MAX_DK, CL_MAX_D);
  const int C = 2 * G * dk + H * dv;
  TL_REQUIRE(C <= width && b_off + (b_off < 0 ? 0 : H) <= width, "channel_chunks: a row of %d is too short", width);
  TL_REQUIRE(taps >= 0 && taps <= CL_MAX_TAPS && (taps == 0 || (conv_w && conv_state && conv_stride >= (long long)(taps - 1) * C)),
             "channel_chunks: a convolution of %d taps without weights, or a block too small", taps);
  TL_REQUIRE(proj && z && state && cu && slots && rec && gam && uf && o, "channel_chunks: a buffer is missing");
  TL_REQUIRE(((uintptr_t)rec | (uintptr_t)gam | (uintptr_t)uf) % 16 == 0, "channel_chunks: a buffer off 16 bytes");
  TL_REQUIRE(stride >= (long long)H * dk * dv, "channel_chunks: a sequence's block is too small");
  const ChunkArgs a{proj, width, 2 * G * dk, z, conv_state, conv_stride, cu, slots, B};
  const ChannelTerms t{G, H, dk, dv, b_off, 0, 0, 0, 0, taps, conv_w, bias, rate, inv_tau, qscale, unit_eps};
  const bool delta = b_off >= 0;
  if (dk <= 64) {
    if (delta) return launch_chunks<64, true>(a, t, chunks, (bf16*)rec, gam, uf, state, stride, o, st);
    return launch_chunks<64, false>(a, t, chunks, (bf16*)rec, gam, uf, state, stride, o, st);
  }
  if (delta) return launch_chunks<128, true>(a, t, chunks, (bf16*)rec, gam, uf, state, stride, o, st);
  return launch_chunks<128, false>(a, t, chunks, (bf16*)rec, gam, uf, state, stride, o, st);
}

}  // extern "C"
