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
// the Delta Rule over Sequence Length).  Three kernels:
//
//   local  one workgroup a chunk and head: convolution, unit norms and decays of its rows, A and B, the solution of
//          the triangular system by blocks of 16 rows, and every operand of the other kernels in the order in which a
//          wave's lanes take it
//   carry  one workgroup 16 columns of a head's state, through the chunks of a sequence in their order, with the state in
//          registers in float.  It leaves the state before every chunk and U, as operands
//   rows   one workgroup a chunk and head: o, the norm over the head and the gate
//
// Decays are kept as logarithms (base 2) summed inside blocks of 16 rows, with the blocks' sums beside them: every
// factor D_i/D_j with i and j in different blocks is then a product of two powers of 2 whose exponents are sums of
// numbers that are none above 0, whatever the decays.  Inside a block the second power has an exponent above 0; a
// block in which some channel decays by more than 2^-STEEP in all is summed in float pair by pair instead.  A float that becomes an
// operand goes in two bfloat16 terms, x = hi + lo (16 bits of its mantissa), and products of two such in three products;
// only operands that nothing but a row's own result depends on (D q and B) are rounded to one.  Sums are float.
#include "channel_linear.hpp"
#include "chunks.hpp"

namespace tl {

constexpr int CC = 64;               // rows of a chunk
constexpr int CC_MAX_DK = 128;
constexpr int FRAG = 512;            // elements of an operand of 16 x 32, lane by lane
constexpr float LOG2E = 1.4426950408889634f;
constexpr float STEEP = 60.f;

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

__device__ __forceinline__ float rcp_(float x) { return __builtin_amdgcn_rcpf(x); }
__device__ __forceinline__ float quick_silu(float a) { return a * rcp_(1.f + ex2(-a * LOG2E)); }
// log2 of a decay (see cl_log_decay) through the exponent and logarithm instructions; log(1 + x) of a small x by its series
__device__ __forceinline__ float quick_softplus(float a) {
  const float x = ex2(-fabsf(a) * LOG2E);
  const float l = x < 0.01f ? x * (1.f - x * (0.5f - x * 0.33333333f)) : __builtin_amdgcn_logf(1.f + x) * 0.69314718f;
  return fmaxf(a, 0.f) + l;
}
__device__ __forceinline__ float log2_decay(float z, bool rated, float rate, float inv_tau) {
  return (rated ? rate * quick_softplus(z) : -quick_softplus(-z) * inv_tau) * LOG2E;
}

// ROWS rows n0 .. of one channel (column c of proj) with the rows that a convolution of at most WIN taps looks back to; rows
// behind `rows` are zeros
template <int ROWS, int WIN> struct ChannelRun {
  float cur[ROWS], win[WIN - 1], w[WIN];
  __device__ __forceinline__ void load(const ChunkArgs& a, const ChannelTerms& t, int C, int n0, int seq_i0, int rows, const float* st, int c) {
    const float* p = a.proj + (size_t)n0 * a.width + c;
#pragma unroll
    for (int r = 0; r < ROWS; ++r) cur[r] = r < rows ? p[(size_t)r * a.width] : 0.f;
    if (!t.taps) return;
#pragma unroll
    for (int j = 0; j < WIN; ++j) {                    // right-aligned: the last is the present row's
      const int back = WIN - 1 - j;
      w[j] = back < t.taps ? t.conv_w[(size_t)c * t.taps + t.taps - 1 - back] : 0.f;
      if (back == 0) continue;
      const int src = seq_i0 - back;
      win[j] = 0.f;
      if (back < t.taps) win[j] = src >= 0 ? p[-(ptrdiff_t)back * a.width] : st[(size_t)(t.taps - 1 + src) * C + c];
    }
  }
  __device__ __forceinline__ void apply(const ChannelTerms& t, int rows) {
    if (!t.taps) return;
#pragma unroll
    for (int r = ROWS - 1; r >= 0; --r) {              // (from the last row up: earlier inputs are still as they were)
      float acc = w[WIN - 1] * cur[r];
#pragma unroll
      for (int back = 1; back < WIN; ++back) acc = fmaf(w[WIN - 1 - back], r >= back ? cur[r >= back ? r - back : 0] : win[r >= back ? 0 : WIN - 1 + r - back], acc);
      cur[r] = r < rows ? quick_silu(acc) : 0.f;
    }
  }
};

template <int DK> constexpr size_t local_lds() {
  return sizeof(float) * (3 * CC * (DK + 4) + 2 * CC * (CC + 4) + 4 * DK + CC + 4 * 16 * 20 + DK / 16);
}

// (I + M) X = X' by blocks of 16 rows for TILES tiles of 16 columns (a lane holds rows 16 I + 4g .. of column m): M below the
// diagonal's blocks, T the inverses of those
template <int TILES>
__device__ __forceinline__ void solve_tiles(f32x4 (&x)[2][4], const float* Ms, int MLD, const float* Ti, int m, int g) {
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  bf16x8 ph[TILES][2], pl[TILES][2];                   // solved blocks 0, 1 and 2, 3 as operands
#pragma unroll
  for (int I = 0; I < 4; ++I) {
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      if (2 * p >= I) continue;
      float mm[8];
      const f32x4 m0 = ld4(Ms + (16 * I + m) * MLD + 32 * p + 4 * g);
      f32x4 m1 = zero;
      if (2 * p + 1 < I) m1 = ld4(Ms + (16 * I + m) * MLD + 32 * p + 16 + 4 * g);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        mm[e] = -m0[e];
        mm[4 + e] = -m1[e];
      }
      bf16x8 mh, ml;
      split8(mm, mh, ml);
#pragma unroll
      for (int k = 0; k < TILES; ++k) {
        x[k][I] = mfma16(mh, ph[k][p], x[k][I]);
        x[k][I] = mfma16(mh, pl[k][p], x[k][I]);
        x[k][I] = mfma16(ml, ph[k][p], x[k][I]);
      }
    }
    bf16x8 th, tl;
    split_tiles(ld4(Ti + (I * 16 + m) * 20 + 4 * g), zero, th, tl);
#pragma unroll
    for (int k = 0; k < TILES; ++k) {
      bf16x8 rh, rl;
      split_tiles(x[k][I], zero, rh, rl);
      f32x4 y = mfma16(th, rh, zero);
      y = mfma16(th, rl, y);
      x[k][I] = mfma16(tl, rh, y);
      if (I == 0) split_tiles(x[k][0], zero, ph[k][0], pl[k][0]);
      if (I == 1) split_tiles(x[k][0], x[k][1], ph[k][0], pl[k][0]);
      if (I == 2) split_tiles(x[k][2], zero, ph[k][1], pl[k][1]);
    }
  }
}

// grid (chunks, H), 4 * DK threads; convolutions of at most WIN taps
template <int DK, bool DELTA, int WIN>
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
  int* steep = reinterpret_cast<int*>(Ti + 4 * 16 * 20);      // [NW]: the wave's channels of its block
  Chunk ch;
  const int c = blockIdx.x, h = blockIdx.y;
  if (!find_chunk(c, a.cu, a.B, CC, ch)) return;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE, m = lane % 16, g = lane / 16;
  const int kh = h / (t.H / t.G), Q = t.G * t.dk, C = 2 * Q + t.H * t.dv;
  const int seq0 = ch.row0 - a.cu[ch.b];             // the chunk's first row counted from the step's first of the sequence
  const float* st = t.taps ? a.conv_state + (long long)a.slots[ch.b] * a.stride : nullptr;
  ChannelRun<4, WIN> vr[4];                          // this wave's first tile of values: rows 16 I + 4g .. of column 16 wave + m
  {
    const int d = tid % DK, i0 = (tid / DK) * 16;
    const int rows = d < t.dk ? ch.rows - i0 : 0, n0 = ch.row0 + i0;
    ChannelRun<16, WIN> xq, xk;
    float z[16];
#pragma unroll
    for (int r = 0; r < 16; ++r) xq.cur[r] = xk.cur[r] = z[r] = 0.f;
    float rate = 0.f, bias = 0.f;
    if (rows > 0) {
      xq.load(a, t, C, n0, seq0 + i0, rows, st, kh * t.dk + d);
      xk.load(a, t, C, n0, seq0 + i0, rows, st, Q + kh * t.dk + d);
      const float* zp = a.z + (size_t)n0 * t.H * t.dk + h * t.dk + d;
#pragma unroll
      for (int r = 0; r < 16; ++r) z[r] = r < rows ? zp[(size_t)r * t.H * t.dk] : 0.f;
      if (t.rate) rate = -expf(t.rate[h]);
      if (t.bias) bias = t.bias[h * t.dk + d];
      xq.apply(t, rows);
      xk.apply(t, rows);
    }
    float sum = 0.f;
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      qs[(i0 + r) * LD + d] = xq.cur[r];
      ks[(i0 + r) * LD + d] = xk.cur[r];
      if (r < rows) sum += log2_decay(z[r] + bias, t.rate != nullptr, rate, t.inv_tau);
      ls[(i0 + r) * LD + d] = sum;
    }
    tot[(tid / DK) * DK + d] = sum;
    const bool any = __any(sum < -STEEP);
    if (lane == 0) steep[wave] = any;
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
  const int vcol = 16 * wave + m;
#pragma unroll
  for (int I = 0; I < 4; ++I) {                        // (fetched now, read behind the products below)
    const int i0 = 16 * I + 4 * g;
#pragma unroll
    for (int r = 0; r < 4; ++r) vr[I].cur[r] = 0.f;
    if (vcol < t.dv && i0 < ch.rows) vr[I].load(a, t, C, ch.row0 + i0, seq0 + i0, ch.rows - i0, st, a.v_off + h * t.dv + vcol);
  }
  __syncthreads();

  // A and B by blocks of 16 x 16
  for (int p = wave; p < 10; p += NW) {
    // pairs (3, 0) .. (3, 3), (2, 0) .. (2, 2), (1, 0), (1, 1), (0, 0)
    const int I = p < 4 ? 3 : (p < 7 ? 2 : (p < 9 ? 1 : 0)), J = p < 4 ? p : (p < 7 ? p - 4 : (p < 9 ? p - 7 : 0));
    bool exact = false;
    if (I == J)
      for (int w = 0; w < DK / WAVE; ++w) exact |= steep[I * (DK / WAVE) + w] != 0;
    f32x4 aa = {0.f, 0.f, 0.f, 0.f}, ab = aa;          // rows 16 I + 4g .., column 16 J + m
    if (!exact) {
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const int d = 32 * s + 8 * g;
        float x[8], q[8], y[8];
#pragma unroll
        for (int q4 = 0; q4 < 2; ++q4) {
          const f32x4 li = ld4(ls + (16 * I + m) * LD + d + 4 * q4), lj = ld4(ls + (16 * J + m) * LD + d + 4 * q4);
          const f32x4 xr = ld4(ks + (16 * I + m) * LD + d + 4 * q4), qr = ld4(qs + (16 * I + m) * LD + d + 4 * q4);
          const f32x4 yr = ld4(ks + (16 * J + m) * LD + d + 4 * q4);
          f32x4 between = -lj;
          for (int M = J; M < I; ++M) between += ld4(tot + M * DK + d + 4 * q4);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const float f = ex2(li[e]);
            x[4 * q4 + e] = xr[e] * f;
            q[4 * q4 + e] = qr[e] * f;
            y[4 * q4 + e] = yr[e] * ex2(between[e]);
          }
        }
        bf16x8 xh, xl, yh, yl;
        split8(y, yh, yl);
        if constexpr (DELTA) {
          split8(x, xh, xl);
          aa = mfma16(xh, yh, aa);
          aa = mfma16(xh, yl, aa);
          aa = mfma16(xl, yh, aa);
        }
        split8(q, xh, xl);
        ab = mfma16(xh, yh, ab);
        ab = mfma16(xh, yl, ab);
        ab = mfma16(xl, yh, ab);
      }
    } else {                                           // pair by pair: this lane's four rows against its column
      for (int d = 0; d < DK; d += 4) {
        const f32x4 y = ld4(ks + (16 * J + m) * LD + d), lj = ld4(ls + (16 * J + m) * LD + d);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = 16 * I + 4 * g + r;
          const f32x4 q = ld4(qs + i * LD + d), x = ld4(ks + i * LD + d), li = ld4(ls + i * LD + d);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const float f = y[e] * ex2(fminf(li[e] - lj[e], 0.f));      // (above 0 only for j > i, which is dropped)
            if constexpr (DELTA) aa[r] = fmaf(x[e], f, aa[r]);
            ab[r] = fmaf(q[e], f, ab[r]);
          }
        }
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * I + 4 * g + r, j = 16 * J + m;
      if constexpr (DELTA) Ms[i * MLD + j] = j < i ? aa[r] * bt[i] : 0.f;
      Bs[i * MLD + j] = j <= i ? ab[r] : 0.f;
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
  bf16* mine = rec + ((size_t)h * gridDim.x + c) * R::FRAGS * FRAG;
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
  if (tid < DK) gam[((size_t)h * gridDim.x + c) * DK + tid] = ex2(tot[tid] + tot[DK + tid] + tot[2 * DK + tid] + tot[3 * DK + tid]);
  __syncthreads();                                     // q has been read: its place takes W

  bf16* w_hi = reinterpret_cast<bf16*>(qs);            // [CC][LD]
  bf16* w_lo = w_hi + CC * LD;
  for (int ct = wave; ct == wave || ct < nct; ct += NW) {        // tile ct of the values and, the first time round, of W
    f32x4 x[2][4];                                     // rows 16 I + 4 g .. of column m
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      const int i0 = 16 * I + 4 * g;
      if (ct != wave) {
        const int col = 16 * ct + m;
#pragma unroll
        for (int r = 0; r < 4; ++r) vr[I].cur[r] = 0.f;
        if (col < t.dv && i0 < ch.rows) vr[I].load(a, t, C, ch.row0 + i0, seq0 + i0, ch.rows - i0, st, a.v_off + h * t.dv + col);
      }
      if (16 * ct + m < t.dv && i0 < ch.rows) vr[I].apply(t, ch.rows - i0);
#pragma unroll
      for (int r = 0; r < 4; ++r) x[0][I][r] = DELTA ? bt[i0 + r] * vr[I].cur[r] : vr[I].cur[r];
    }
    if constexpr (DELTA) {
      if (ct == wave) {
        const int d = 16 * ct + m;
        float before = 0.f;
#pragma unroll
        for (int I = 0; I < 4; ++I) {
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int i = 16 * I + 4 * g + r;
            x[1][I][r] = bt[i] * ks[i * LD + d] * ex2(before + ls[i * LD + d]);
          }
          before += tot[I * DK + d];
        }
        solve_tiles<2>(x, Ms, MLD, Ti, m, g);
#pragma unroll
        for (int I = 0; I < 4; ++I)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int at = (16 * I + 4 * g + r) * LD + d;
            const float v = -x[1][I][r];
            const bf16 hi = (bf16)v;
            w_hi[at] = hi;
            w_lo[at] = (bf16)(v - (float)hi);
          }
      } else {
        solve_tiles<1>(x, Ms, MLD, Ti, m, g);
      }
    }
    if (ct < nct) {
      float* up = uf + (((size_t)h * gridDim.x + c) * nct + ct) * (CC * 16);
#pragma unroll
      for (int I = 0; I < 4; ++I) *reinterpret_cast<f32x4*>(up + (I * WAVE + lane) * 4) = x[0][I];
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

// what `carry` leaves for a tile of 16 columns of a chunk and head, in FRAGs: the state before the chunk, hi and lo
// [DK/32][2], and U, hi and lo [2][2]
template <int DK> struct Carried {
  static constexpr int U = DK / 16, FRAGS = U + 4;
};
constexpr int XCDS = 8;              // parts of the chip with a second-level cache each; workgroups go round them in turn

// 1 KB from memory straight into LDS: lane l's 16 bytes at p to dst + 16 l
__device__ __forceinline__ void bring(const void* p, void* dst) {
  __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)p, (__attribute__((address_space(3))) void*)dst, 16, 0, 0);
}
template <int N> __device__ __forceinline__ void wait_all_but() {       // until at most N accesses to memory are under way
  asm volatile("s_waitcnt vmcnt(%0)" ::"n"(N) : "memory");
}
__device__ __forceinline__ void wait_lds() { asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory"); }

// a chunk's place in the ring of `carry`, in KB: W (hi, lo), (D_last/D k)^T (hi, lo), the tile's values, D_last; and, behind the
// ring, what the waves hand each other: the state (hi, lo) and U (hi, lo) as operands
template <int DK, bool DELTA> struct Ring {
  static constexpr int W = 0, K = DELTA ? DK / 4 : 0, U = K + DK / 4, G = U + 4, SLOT = (G + 1) * 1024;
  static constexpr int SLOTS = SLOT > 48 * 1024 ? 2 : 3;
  static constexpr int S_OUT = SLOTS * SLOT, U_OUT = S_OUT + DK / 16 * 1024, BYTES = U_OUT + 4 * 1024;
};

// One workgroup a tile of 16 columns of a head's state; the tiles of a head lie on one part of the chip, where they share
// what they read.  Wave w keeps rows 32 w .. 32 w + 31 of the state (in its registers, in float) and works out its share of the
// chunk's 64 rows of U; the waves hand each other the state and U through LDS, a barrier each.  Operands come
// through a ring in LDS, SLOTS chunks ahead, in two groups a chunk, each issued once the group it replaces has been read.  A
// wave's accesses complete in their order: it waits until no more are under way than it has issued behind the group (its own
// share of it; the barrier covers the others'), and behind the last chunk the last one's operands are fetched again, so that
// the count holds.  grid (XCDS * ceil(H / XCDS) * nct, B), DK / 32 waves
template <int DK, bool DELTA>
__global__ void __launch_bounds__(2 * DK)
channel_carry_kernel(const bf16* __restrict__ rec, const float* __restrict__ gam, const float* __restrict__ uf, int nct, int total, int H, int dk,
                     int dv, float* __restrict__ state, long long stride, const int* __restrict__ cu, const int* __restrict__ slots,
                     bf16* __restrict__ su) {
  using R = Record<DK, DELTA>;
  using S_ = Carried<DK>;
  using L = Ring<DK, DELTA>;
  constexpr int KS = DK / 32, NS = L::SLOTS, RI = 4 / KS;        // RI: blocks of 16 rows of U a wave
  constexpr int G1 = (DELTA ? 8 : 0) + RI + 1, G2 = 8, BEHIND = (NS - 1) * (G1 + G2);
  extern __shared__ __attribute__((aligned(1024))) unsigned char ring[];
  const int idx = blockIdx.x / XCDS, h = blockIdx.x % XCDS + XCDS * (idx / nct), ct = idx % nct, b = blockIdx.y;
  if (h >= H) return;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE, m = lane % 16, g = lane / 16, col = 16 * ct + m;
  int first = 0;
  for (int s = 0; s < b; ++s) first += (cu[s + 1] - cu[s] + CC - 1) / CC;
  const int n = cu[b + 1] - cu[b], chunks = (n + CC - 1) / CC;
  if (chunks == 0) return;
  const bool ok = col < dv;
  float* S_g = state + (long long)slots[b] * stride + ((size_t)h * dv + (ok ? col : 0)) * dk;
  f32x4 S[2];                                          // rows 32 wave + 16 t + 4g .. of column m
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 32 * wave + 16 * t + 4 * g + r;
      S[t][r] = ok && d < dk ? S_g[d] : 0.f;
    }
  // group 1 of a chunk: W, the values, D_last; group 2: (D_last/D k)^T.  Every wave its share (D_last: each, the same)
  auto issue1 = [&](int c) {
    const size_t at = (size_t)h * total + first + min(c, chunks - 1);
    unsigned char* slot = ring + (c % NS) * L::SLOT;
    if constexpr (DELTA) {
      const bf16* p = rec + (at * R::FRAGS + R::W_HI + 8 * wave) * FRAG + lane * 8;
#pragma unroll
      for (int f = 0; f < 8; ++f) bring(p + f * FRAG, slot + (L::W + 8 * wave + f) * 1024);
    }
    const float* up = uf + (at * nct + ct) * (CC * 16) + RI * wave * WAVE * 4 + lane * 4;
#pragma unroll
    for (int I = 0; I < RI; ++I) bring(up + I * WAVE * 4, slot + (L::U + RI * wave + I) * 1024);
    bring(gam + at * DK + (lane * 4) % DK, slot + L::G * 1024);
  };
  auto issue2 = [&](int c) {
    const size_t at = (size_t)h * total + first + min(c, chunks - 1);
    const bf16* p = rec + (at * R::FRAGS + R::K_HI + 8 * wave) * FRAG + lane * 8;
    unsigned char* slot = ring + (c % NS) * L::SLOT;
#pragma unroll
    for (int f = 0; f < 8; ++f) bring(p + f * FRAG, slot + (L::K + 8 * wave + f) * 1024);
  };
  for (int c = 0; c < NS; ++c) {
    issue1(c);
    if (c + 1 < NS) issue2(c);
  }
  bf16* sp = su + (((size_t)h * total + first) * nct + ct) * S_::FRAGS * FRAG + lane * 8;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  for (int c = 0; c < chunks; ++c) {
    const unsigned char* slot = ring + (c % NS) * L::SLOT;
    auto frag = [&](const unsigned char* p) { return *reinterpret_cast<const bf16x8*>(p + lane * 16); };
    bf16x8 hi, lo;
    split_tiles(S[0], S[1], hi, lo);                   // this wave's rows of the state as an operand
    if constexpr (DELTA) {
      *reinterpret_cast<bf16x8*>(ring + L::S_OUT + (2 * wave) * 1024 + lane * 16) = hi;
      *reinterpret_cast<bf16x8*>(ring + L::S_OUT + (2 * wave + 1) * 1024 + lane * 16) = lo;
    }
    wait_all_but<BEHIND>();
    wait_lds();
    __builtin_amdgcn_s_barrier();                      // group 1 and every wave's state are there; the last group 2 has been read
    issue2(c + NS - 1);
    *reinterpret_cast<bf16x8*>(sp + (size_t)(2 * wave) * FRAG) = hi;
    *reinterpret_cast<bf16x8*>(sp + (size_t)(2 * wave + 1) * FRAG) = lo;
    f32x4 gn[2];
#pragma unroll
    for (int t = 0; t < 2; ++t) gn[t] = *reinterpret_cast<const f32x4*>(slot + L::G * 1024 + (32 * wave + 16 * t + 4 * g) * 4);
    f32x4 u[RI], u1[RI], u2[RI];
#pragma unroll
    for (int I = 0; I < RI; ++I) {
      u[I] = *reinterpret_cast<const f32x4*>(slot + (L::U + RI * wave + I) * 1024 + lane * 16);
      u1[I] = u2[I] = zero;
    }
    if constexpr (DELTA) {
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const bf16x8 sh = frag(ring + L::S_OUT + (2 * s) * 1024), sl = frag(ring + L::S_OUT + (2 * s + 1) * 1024);
#pragma unroll
        for (int I = 0; I < RI; ++I) {
          const int f = (RI * wave + I) * KS + s;
          const bf16x8 wh = frag(slot + (L::W + f) * 1024), wl = frag(slot + (L::W + 4 * KS + f) * 1024);
          u[I] = mfma16(wh, sh, u[I]);
          u1[I] = mfma16(wh, sl, u1[I]);
          u2[I] = mfma16(wl, sh, u2[I]);
        }
      }
    }
#pragma unroll
    for (int I = 0; I < RI; ++I) {                     // this wave's rows of U, half of an operand each
      const f32x4 x = u[I] + (u1[I] + u2[I]);
      const int at = RI * wave + I, p = (S_::U + 2 * (at / 2)) * FRAG + (at % 2) * 4, q = L::U_OUT + 2 * (at / 2) * 1024 + (at % 2) * 8;
      bf16x4 uh, ul;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        uh[r] = (bf16)x[r];
        ul[r] = (bf16)(x[r] - (float)uh[r]);
      }
      *reinterpret_cast<bf16x4*>(ring + q + lane * 16) = uh;
      *reinterpret_cast<bf16x4*>(ring + q + 1024 + lane * 16) = ul;
      *reinterpret_cast<bf16x4*>(sp + p) = uh;
      *reinterpret_cast<bf16x4*>(sp + p + FRAG) = ul;
    }
    wait_all_but<BEHIND>();
    wait_lds();
    __builtin_amdgcn_s_barrier();                      // group 2 and every wave's U are there; group 1 has been read
    issue1(c + NS);
    f32x4 lowS[2];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      S[t] *= gn[t];
      lowS[t] = zero;
    }
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const bf16x8 uh = frag(ring + L::U_OUT + (2 * s) * 1024), ul = frag(ring + L::U_OUT + (2 * s + 1) * 1024);
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        const int f = 2 * (2 * wave + t) + s;
        const bf16x8 kh = frag(slot + (L::K + f) * 1024), kl = frag(slot + (L::K + DK / 8 + f) * 1024);
        S[t] = mfma16(kh, uh, S[t]);
        lowS[t] = mfma16(kh, ul, lowS[t]);
        lowS[t] = mfma16(kl, uh, lowS[t]);
      }
    }
#pragma unroll
    for (int t = 0; t < 2; ++t) S[t] += lowS[t];
    sp += (size_t)nct * S_::FRAGS * FRAG;
  }
  wait_all_but<0>();                                   // (nothing may arrive in LDS behind the wave's end)
  if (!ok) return;
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 32 * wave + 16 * t + 4 * g + r;
      if (d < dk) S_g[d] = S[t][r];
    }
}

struct RowsOut {
  const float* w;            // [dv] (null: no weight)
  const float* gate;         // the gate's first column in rows `gate_stride` apart
  int gate_stride, gate_silu;
  float eps, factor;
  bf16* out;                 // rows `out_stride` apart
  int out_stride;
};
constexpr int RW_NT = 512, RW_TILES = 2;      // threads; tiles of 16 columns a wave at most (dv up to 256)

// out = factor * rms(o) * w * gate with o = (D q) S + B U.  grid (chunks, H)
template <int DK, bool DELTA>
__global__ void __launch_bounds__(RW_NT)
channel_out_kernel(const bf16* __restrict__ rec, const bf16* __restrict__ su, int nct, int H, int dv, const int* __restrict__ cu, int B,
                   RowsOut z) {
  using R = Record<DK, DELTA>;
  using S_ = Carried<DK>;
  constexpr int KS = DK / 32, NW = RW_NT / WAVE;
  extern __shared__ __attribute__((aligned(16))) unsigned char rw_lds[];
  const int ld = 16 * nct + 8;
  bf16* os = reinterpret_cast<bf16*>(rw_lds);                            // [CC][ld]
  float* sums = reinterpret_cast<float*>(os + CC * ld);                   // [NW][CC]
  Chunk ch;
  const int c = blockIdx.x, h = blockIdx.y;
  if (!find_chunk(c, cu, B, CC, ch)) return;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid % WAVE, m = lane % 16, g = lane / 16;
  const bf16* mine = rec + ((size_t)h * gridDim.x + c) * R::FRAGS * FRAG + lane * 8;
  const bf16* sp = su + ((size_t)h * gridDim.x + c) * nct * S_::FRAGS * FRAG + lane * 8;
  auto frag = [&](const bf16* p, int f) { return *reinterpret_cast<const bf16x8*>(p + (size_t)f * FRAG); };
  f32x4 o[RW_TILES][4], gt[RW_TILES][4];
  f32x4 ss[4];
#pragma unroll
  for (int k = 0; k < RW_TILES; ++k) {                 // the gates, fetched ahead
    const int col = 16 * (wave + k * NW) + m;
#pragma unroll
    for (int I = 0; I < 4; ++I)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * I + 4 * g + r;
        gt[k][I][r] = col < dv && i < ch.rows ? z.gate[(size_t)(ch.row0 + i) * z.gate_stride + (size_t)h * dv + col] : 0.f;
      }
  }
#pragma unroll
  for (int I = 0; I < 4; ++I) ss[I] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int k = 0; k < RW_TILES; ++k) {
    const int ct = wave + k * NW;
    if (ct >= nct) break;
    const bf16* tp = sp + (size_t)ct * S_::FRAGS * FRAG;
#pragma unroll
    for (int I = 0; I < 4; ++I) o[k][I] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const bf16x8 sh = frag(tp, 2 * s), sl = frag(tp, 2 * s + 1);
#pragma unroll
      for (int I = 0; I < 4; ++I) {
        const bf16x8 q = frag(mine, R::Q + I * KS + s);
        o[k][I] = mfma16(q, sh, o[k][I]);
        o[k][I] = mfma16(q, sl, o[k][I]);
      }
    }
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const bf16x8 uh = frag(tp, S_::U + 2 * s), ul = frag(tp, S_::U + 2 * s + 1);
#pragma unroll
      for (int I = 2 * s; I < 4; ++I) {                // (B is zero above the diagonal)
        const bf16x8 bb = frag(mine, R::B + 2 * I + s);
        o[k][I] = mfma16(bb, uh, o[k][I]);
        o[k][I] = mfma16(bb, ul, o[k][I]);
      }
    }
#pragma unroll
    for (int I = 0; I < 4; ++I) ss[I] += o[k][I] * o[k][I];      // (columns behind dv are zeros)
  }
#pragma unroll
  for (int I = 0; I < 4; ++I)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float sum = row16_sum(ss[I][r]);
      if (m == 0) sums[wave * CC + 16 * I + 4 * g + r] = sum;
    }
  __syncthreads();
#pragma unroll
  for (int I = 0; I < 4; ++I)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      float sum = 0.f;
#pragma unroll
      for (int w = 0; w < NW; ++w) sum += sums[w * CC + 16 * I + 4 * g + r];
      ss[I][r] = z.factor / sqrtf(sum / (float)dv + z.eps);
    }
#pragma unroll
  for (int k = 0; k < RW_TILES; ++k) {
    const int ct = wave + k * NW, col = 16 * ct + m;
    if (ct >= nct) break;
    if (col >= dv) continue;
    const float wc = z.w ? z.w[col] : 1.f;
#pragma unroll
    for (int I = 0; I < 4; ++I)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * I + 4 * g + r;
        if (i >= ch.rows) continue;
        const float a = gt[k][I][r];
        os[i * ld + col] = (bf16)(o[k][I][r] * ss[I][r] * wc * ((z.gate_silu ? a : 1.f) * rcp_(1.f + ex2(-a * LOG2E))));
      }
  }
  __syncthreads();
  bf16* out = z.out + (size_t)ch.row0 * z.out_stride + (size_t)h * dv;
  if (dv % 8 == 0 && z.out_stride % 8 == 0 && (uintptr_t)z.out % 16 == 0) {
    const int per = dv / 8;
    for (int e = tid; e < ch.rows * per; e += RW_NT) {
      const int i = e / per, col = (e % per) * 8;
      *reinterpret_cast<bf16x8*>(out + (size_t)i * z.out_stride + col) = *reinterpret_cast<const bf16x8*>(os + i * ld + col);
    }
  } else {
    for (int e = tid; e < ch.rows * dv; e += RW_NT) out[(size_t)(e / dv) * z.out_stride + e % dv] = os[(e / dv) * ld + e % dv];
  }
}

template <int DK, bool DELTA, int WIN>
static int launch_local(const ChunkArgs& a, const ChannelTerms& t, int chunks, bf16* rec, float* gam, float* uf, int nct, hipStream_t st) {
  static bool raised = false;
  if (!raised) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&channel_local_kernel<DK, DELTA, WIN>),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)local_lds<DK>());
    if (e != hipSuccess) {
      set_error("channel_chunks: cannot have %zu bytes of LDS: %s", local_lds<DK>(), hipGetErrorString(e));
      return 2;
    }
    raised = true;
  }
  channel_local_kernel<DK, DELTA, WIN><<<dim3(chunks, t.H), 4 * DK, local_lds<DK>(), st>>>(a, t, rec, gam, uf, nct);
  TL_LAUNCH_CHECK("channel_local");
  return 0;
}

template <int DK, bool DELTA>
static int launch_chunks(const ChunkArgs& a, const ChannelTerms& t, int chunks, bf16* rec, float* gam, float* uf, bf16* su, float* state,
                         long long stride, const RowsOut& z, hipStream_t st) {
  const int nct = (t.dv + 15) / 16;
  const int rc = t.taps <= 4 ? launch_local<DK, DELTA, 4>(a, t, chunks, rec, gam, uf, nct, st)
                             : launch_local<DK, DELTA, CL_MAX_TAPS>(a, t, chunks, rec, gam, uf, nct, st);
  if (rc) return rc;
  constexpr int ring = Ring<DK, DELTA>::BYTES;
  static bool raised = false;
  if (!raised) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&channel_carry_kernel<DK, DELTA>),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, ring);
    if (e != hipSuccess) {
      set_error("channel_chunks: cannot have %d bytes of LDS: %s", ring, hipGetErrorString(e));
      return 2;
    }
    raised = true;
  }
  channel_carry_kernel<DK, DELTA><<<dim3(XCDS * ((t.H + XCDS - 1) / XCDS) * nct, a.B), 2 * DK, ring, st>>>(rec, gam, uf, nct, chunks, t.H, t.dk,
                                                                                                        t.dv, state, stride, a.cu, a.slots, su);
  TL_LAUNCH_CHECK("channel_carry");
  const size_t lds = (size_t)CC * (16 * nct + 8) * sizeof(bf16) + (RW_NT / WAVE) * CC * sizeof(float);
  channel_out_kernel<DK, DELTA><<<dim3(chunks, t.H), RW_NT, lds, st>>>(rec, su, nct, t.H, t.dv, a.cu, a.B, z);
  TL_LAUNCH_CHECK("channel_out");
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
// bfloat16 elements that `carry` leaves for a tile of 16 columns of a chunk and head
int tl_channel_carried(int dk) { return (dk <= 64 ? Carried<64>::FRAGS : Carried<128>::FRAGS) * FRAG; }

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
// chunks.  Scratch: rec chunks*H*tl_channel_record, gam chunks*H*tl_channel_padded floats, uf chunks*H*ceil(dv/16)*1024 floats, su
// chunks*H*ceil(dv/16)*tl_channel_carried.  out bfloat16 [n, H*dv] = factor * rms(o) * w * (silu or logistic of gate).
int tl_channel_chunks(const float* proj, int width, int G, int H, int dk, int dv, int b_off, int taps, const float* conv_w, const float* bias,
                      const float* rate, float inv_tau, float qscale, float unit_eps, const float* z, const float* conv_state,
                      long long conv_stride, float* state, long long stride, const int* cu, const int* slots, int n, int B, int chunks,
                      void* rec, float* gam, float* uf, void* su, const float* w, const float* gate, int gate_stride, int gate_silu,
                      float eps, float factor, void* out, int out_stride, hipStream_t st) {
  TL_REQUIRE(n > 0 && B > 0 && B <= 65535 && G > 0 && H > 0 && H <= 65535 && H % G == 0 && chunks > 0, "channel_chunks: bad sizes n=%d B=%d G=%d H=%d chunks=%d",
             n, B, G, H, chunks);
  TL_REQUIRE(dk > 0 && dk <= CC_MAX_DK && dv > 0 && dv <= CL_MAX_D, "channel_chunks: heads of %d and %d are not served (up to %d and %d)", dk, dv,
             CC_MAX_DK, CL_MAX_D);
  const int C = 2 * G * dk + H * dv;
  TL_REQUIRE(C <= width && b_off + (b_off < 0 ? 0 : H) <= width, "channel_chunks: a row of %d is too short", width);
  TL_REQUIRE(taps >= 0 && taps <= CL_MAX_TAPS && (taps == 0 || (conv_w && (conv_state || taps == 1) && conv_stride >= (long long)(taps - 1) * C)),
             "channel_chunks: a convolution of %d taps without weights, or a block too small", taps);
  TL_REQUIRE(proj && z && state && cu && slots && rec && gam && uf && su && gate && out, "channel_chunks: a buffer is missing");
  TL_REQUIRE(((uintptr_t)rec | (uintptr_t)gam | (uintptr_t)uf | (uintptr_t)su) % 16 == 0, "channel_chunks: a buffer off 16 bytes");
  TL_REQUIRE(stride >= (long long)H * dk * dv, "channel_chunks: a sequence's block is too small");
  TL_REQUIRE(gate_stride >= H * dv && out_stride >= H * dv, "channel_chunks: rows of the gate or the result are too short");
  const ChunkArgs a{proj, width, 2 * G * dk, z, conv_state, conv_stride, cu, slots, B};
  const ChannelTerms t{G, H, dk, dv, b_off, 0, 0, 0, 0, taps, conv_w, bias, rate, inv_tau, qscale, unit_eps};
  const RowsOut r{w, gate, gate_stride, gate_silu, eps, factor, (bf16*)out, out_stride};
  const bool delta = b_off >= 0;
  if (dk <= 64) {
    if (delta) return launch_chunks<64, true>(a, t, chunks, (bf16*)rec, gam, uf, (bf16*)su, state, stride, r, st);
    return launch_chunks<64, false>(a, t, chunks, (bf16*)rec, gam, uf, (bf16*)su, state, stride, r, st);
  }
  if (delta) return launch_chunks<128, true>(a, t, chunks, (bf16*)rec, gam, uf, (bf16*)su, state, stride, r, st);
  return launch_chunks<128, false>(a, t, chunks, (bf16*)rec, gam, uf, (bf16*)su, state, stride, r, st);
}

}  // extern "C"
