// Retention by chunks of rows on the matrix cores: bfloat16 steps that bring many rows (see
// retention.hip for the mechanism).  A sequence's new rows are cut into chunks of RC = 256 counted
// from the step's first row; with i, j the places in a chunk of L rows and S the state before it,
//
//   o_i = decay^(i+1) S^T q_i + sum_{j <= i} decay^(i-j) (k_j . q_i) v_j
//   S  <- decay^L S + sum_j decay^(L-1-j) k_j v_j^T
//
// Four kernels:
//   prepare  q and k rotated (k times its factor) as rows; k times decay^(L-1-j) and v transposed, chunk by chunk
//   states   what every chunk adds to the state, [dk, dv] in float: a product over the chunk's rows
//   carry    the chunks of a sequence in their order, element by element of the state in float: leaves the state
//            before every chunk, transposed, and the last one in the sequence's block
//   rows     128 rows of a chunk and one head a workgroup: the state's part, then the chunk's keys up to the rows,
//            the norm over the head and the gate
// A float that becomes an operand of a product beside the plain rows of q, k and v (the decayed k, the
// state, the decayed weights of the keys) goes in two bfloat16 terms, x = hi + lo, which carry 16 bits
// of its mantissa; the sums are float.
#include "chunks.hpp"
#include "common.hpp"

namespace tl {

constexpr int RC = 256;              // rows of a chunk
constexpr int RC_TILE = 64;          // rows that a workgroup of `prepare` takes
constexpr int RC_MAX_D = 256;

__device__ __forceinline__ bf16x8 rld8(const bf16* p) { return *reinterpret_cast<const bf16x8*>(p); }
__device__ __forceinline__ bf16x4 rld4(const bf16* p) { return *reinterpret_cast<const bf16x4*>(p); }
__device__ __forceinline__ bf16x8 rz8() {
  bf16x8 z;
#pragma unroll
  for (int i = 0; i < 8; ++i) z[i] = (bf16)0.f;
  return z;
}

// grid (chunks * RC / RC_TILE, H)
__global__ void __launch_bounds__(256)
retention_prepare_kernel(const float* __restrict__ proj, int width, int H, int dk, int dv, const int* __restrict__ row_pos,
                         Rotation rot, float kscale, const float* __restrict__ log2_decay, const int* __restrict__ cu, int B,
                         bf16* __restrict__ q, bf16* __restrict__ k, bf16* __restrict__ kt_hi, bf16* __restrict__ kt_lo,
                         bf16* __restrict__ vt) {
  extern __shared__ float rc_lds[];                    // [RC_TILE][max(dk, 64) + 1]
  Chunk ch;
  const int c = blockIdx.x / (RC / RC_TILE), t0 = (blockIdx.x % (RC / RC_TILE)) * RC_TILE, h = blockIdx.y, t = threadIdx.x;
  if (!find_chunk(c, cu, B, RC, ch) || t0 >= ch.rows) return;
  const int rows = min(RC_TILE, ch.rows - t0), n0 = ch.row0 + t0, ld = dk + 1;
  const int half = rot.rotary_dim / 2, units = dk - half;        // a rotated pair, or a channel behind them
  for (int e = t; e < RC_TILE * units; e += 256) {
    const int i = e / units, u = e % units;
    if (i >= rows) {                                   // (columns behind the chunk's last row are zeros)
      if (u < half) {
        int a, d;
        pair_channels(u, rot.rotary_dim, rot.interleaved, a, d);
        rc_lds[i * ld + a] = rc_lds[i * ld + d] = 0.f;
      } else {
        rc_lds[i * ld + half + u] = 0.f;
      }
      continue;
    }
    const float* qr = proj + (size_t)(n0 + i) * width + (size_t)h * dk;
    const float* kr = qr + (size_t)H * dk;
    bf16* qo = q + ((size_t)(n0 + i) * H + h) * dk;
    bf16* ko = k + ((size_t)(n0 + i) * H + h) * dk;
    if (u < half) {
      int a, d;
      pair_channels(u, rot.rotary_dim, rot.interleaved, a, d);
      float sn, cs, x, y;
      sincosf((float)row_pos[n0 + i] * rot.inv_freq[u], &sn, &cs);
      cs *= rot.magnitude;
      sn *= rot.magnitude;
      rotate_pair(qr[a], qr[d], cs, sn, x, y);
      qo[a] = (bf16)x;
      qo[d] = (bf16)y;
      rotate_pair(kr[a], kr[d], cs, sn, x, y);
      x *= kscale;
      y *= kscale;
      ko[a] = (bf16)x;
      ko[d] = (bf16)y;
      rc_lds[i * ld + a] = x;
      rc_lds[i * ld + d] = y;
    } else {
      const int a = half + u;                          // (2 half + the (u - half)-th channel behind the pairs)
      qo[a] = (bf16)qr[a];
      const float x = kr[a] * kscale;
      ko[a] = (bf16)x;
      rc_lds[i * ld + a] = x;
    }
  }
  __syncthreads();
  const float lg = log2_decay[h];
  const size_t head = (size_t)c * H + h;
  for (int e = t; e < dk * RC_TILE; e += 256) {
    const int d = e / RC_TILE, i = e % RC_TILE;
    // rows behind the chunk's last: zeros, whatever the factor (its exponent is cut off at 0)
    const float x = rc_lds[i * ld + d] * exp2f((float)max(ch.rows - 1 - t0 - i, 0) * lg);
    const bf16 hi = (bf16)x;
    const size_t at = (head * dk + d) * RC + t0 + i;
    kt_hi[at] = hi;
    kt_lo[at] = (bf16)(x - (float)hi);
  }
  for (int d0 = 0; d0 < dv; d0 += RC_TILE) {
    const int m = min(RC_TILE, dv - d0);
    __syncthreads();
    for (int e = t; e < RC_TILE * RC_TILE; e += 256) {
      const int i = e / RC_TILE, d = e % RC_TILE;
      if (d < m)
        rc_lds[i * (RC_TILE + 1) + d] =
            i < rows ? proj[(size_t)(n0 + i) * width + (size_t)2 * H * dk + (size_t)h * dv + d0 + d] : 0.f;
    }
    __syncthreads();
    for (int e = t; e < m * RC_TILE; e += 256) {
      const int d = e / RC_TILE, i = e % RC_TILE;
      vt[(head * dv + d0 + d) * RC + t0 + i] = (bf16)rc_lds[i * (RC_TILE + 1) + d];
    }
  }
}

// kv[c, h] [dk, dv] = sum_j (decayed k_j) v_j^T: a workgroup a tile of 64 x 64, a wave 32 x 32.  grid (chunks, H, tiles)
__global__ void __launch_bounds__(256)
retention_states_kernel(const bf16* __restrict__ kt_hi, const bf16* __restrict__ kt_lo, const bf16* __restrict__ vt, int H, int dk,
                        int dv, const int* __restrict__ cu, int B, float* __restrict__ kv) {
  Chunk ch;
  const int c = blockIdx.x, h = blockIdx.y, nt = (dv + 63) / 64;
  if (!find_chunk(c, cu, B, RC, ch)) return;
  const int wave = threadIdx.x / 64, lane = threadIdx.x % 64, l32 = lane % 32, half = lane / 32;
  const int m0 = (blockIdx.z / nt) * 64 + (wave / 2) * 32, n0 = (blockIdx.z % nt) * 64 + (wave % 2) * 32;
  if (m0 >= dk || n0 >= dv) return;
  const size_t head = (size_t)c * H + h;
  const size_t ka = (head * dk + min(m0 + l32, dk - 1)) * RC + 8 * half, va = (head * dv + min(n0 + l32, dv - 1)) * RC + 8 * half;
  f32x16 acc;
#pragma unroll
  for (int r = 0; r < 16; ++r) acc[r] = 0.f;
  const int steps = (ch.rows + RC_TILE - 1) / RC_TILE * (RC_TILE / 16);       // (whole tiles: `prepare` has filled them with zeros)
#pragma unroll 4
  for (int s = 0; s < steps; ++s) {
    const bf16x8 v = rld8(vt + va + s * 16);
    acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(rld8(kt_hi + ka + s * 16), v, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(rld8(kt_lo + ka + s * 16), v, acc, 0, 0, 0);
  }
  if (n0 + l32 >= dv) return;
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    const int m = m0 + 8 * (r / 4) + 4 * half + (r % 4);
    if (m < dk) kv[(head * dk + m) * dv + n0 + l32] = acc[r];
  }
}

// A tile of 32 x 32 of a head's state through the chunks of one sequence: st_hi/st_lo [chunk, H, dv, dk] = the state
// before the chunk.  grid (tiles, H, B)
__global__ void __launch_bounds__(256)
retention_carry_kernel(const float* __restrict__ kv, int H, int dk, int dv, const float* __restrict__ log2_decay,
                       float* __restrict__ state, long long stride, const int* __restrict__ cu, const int* __restrict__ slots,
                       bf16* __restrict__ st_hi, bf16* __restrict__ st_lo) {
  __shared__ float tile[32][33];
  const int h = blockIdx.y, b = blockIdx.z, t = threadIdx.x;
  const int nt = (dv + 31) / 32, i0 = (blockIdx.x / nt) * 32, j0 = (blockIdx.x % nt) * 32;
  int first = 0;
  for (int s = 0; s < b; ++s) first += (cu[s + 1] - cu[s] + RC - 1) / RC;
  const int n = cu[b + 1] - cu[b], chunks = (n + RC - 1) / RC;
  if (chunks == 0) return;
  const int j = t % 32, ii = t / 32;                   // this thread: rows ii, ii + 8, .. of column j
  float* S_g = state + (long long)slots[b] * stride + (size_t)h * dk * dv;
  const float lg = log2_decay[h];
  float S[4], nxt[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int i = i0 + ii + 8 * r;
    const bool ok = i < dk && j0 + j < dv;
    S[r] = ok ? S_g[(size_t)i * dv + j0 + j] : 0.f;
    nxt[r] = ok ? kv[(((size_t)first * H + h) * dk + i) * dv + j0 + j] : 0.f;
  }
  for (int c = 0; c < chunks; ++c) {
    const size_t head = (size_t)(first + c) * H + h;
    float cur[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      cur[r] = nxt[r];
      const int i = i0 + ii + 8 * r;
      if (c + 1 < chunks && i < dk && j0 + j < dv) nxt[r] = kv[((head + H) * dk + i) * dv + j0 + j];
    }
    __syncthreads();
#pragma unroll
    for (int r = 0; r < 4; ++r) tile[ii + 8 * r][j] = S[r];
    __syncthreads();
#pragma unroll
    for (int r = 0; r < 4; ++r) {                      // transposed: consecutive threads along dk
      const int jj = ii + 8 * r, i = j;
      if (i0 + i < dk && j0 + jj < dv) {
        const float x = tile[i][jj];
        const bf16 hi = (bf16)x;
        const size_t at = (head * dv + j0 + jj) * dk + i0 + i;
        st_hi[at] = hi;
        st_lo[at] = (bf16)(x - (float)hi);
      }
    }
    const float f = exp2f((float)min(RC, n - c * RC) * lg);
#pragma unroll
    for (int r = 0; r < 4; ++r) S[r] = fmaf(f, S[r], cur[r]);
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int i = i0 + ii + 8 * r;
    if (i < dk && j0 + j < dv) S_g[(size_t)i * dv + j0 + j] = S[r];
  }
}

// out[row, h] = rms(o) * silu(g).  grid (2 * chunks, H): 128 rows of a chunk, a wave 32 of them.  As in the attention
// kernels a lane owns one row's column of the transposed products S^T = K Q^T and O^T = V^T P^T.
constexpr int RR_BM = 128, RR_BN = 64, RR_VLD = RR_BN + 4;

template <int DK, int DV>
__global__ void __launch_bounds__(256, DK + DV <= 256 ? 2 : 1)
retention_rows_kernel(const bf16* __restrict__ q, const bf16* __restrict__ k, const bf16* __restrict__ vt,
                      const bf16* __restrict__ st_hi, const bf16* __restrict__ st_lo, const float* __restrict__ gate, int gate_stride,
                      int H, int dk, int dv, const float* __restrict__ log2_decay, float eps, const int* __restrict__ cu, int B,
                      bf16* __restrict__ out) {
  constexpr int KB = DK / 16, VB = DV / 32, KLD = DK + 8, CH = DK / 8;
  extern __shared__ __attribute__((aligned(16))) unsigned char rr_smem[];
  bf16* Ks = reinterpret_cast<bf16*>(rr_smem);         // [RR_BN][KLD]
  bf16* Vt = Ks + RR_BN * KLD;                         // [DV][RR_VLD]
  Chunk ch;
  // the second half of a chunk has the longer way: it goes first
  const int c = blockIdx.x / 2, q0 = (1 - (int)(blockIdx.x % 2)) * RR_BM, h = blockIdx.y;
  if (!find_chunk(c, cu, B, RC, ch) || q0 >= ch.rows) return;
  const int tid = threadIdx.x, wave = tid / 64, lane = tid % 64, l32 = lane % 32, half = lane / 32;
  const int i = q0 + wave * 32 + l32;                  // this lane's row in the chunk
  const bool ok = i < ch.rows;
  const int wi_lo = q0 + wave * 32, wi_hi = wi_lo + 31;
  const int row = ch.row0 + min(i, ch.rows - 1);
  const float lg = log2_decay[h];
  const size_t head = (size_t)c * H + h;

  bf16x8 qreg[KB];
  {
    const bf16* qp = q + ((size_t)row * H + h) * dk;
#pragma unroll
    for (int kb = 0; kb < KB; ++kb) {
      const int e = kb * 16 + 8 * half;
      qreg[kb] = (e + 8 <= dk) ? rld8(qp + e) : rz8();
    }
  }
  f32x16 o[VB];
#pragma unroll
  for (int vb = 0; vb < VB; ++vb) {
#pragma unroll
    for (int r = 0; r < 16; ++r) o[vb][r] = 0.f;
    const size_t at = (head * dv + min(vb * 32 + l32, dv - 1)) * dk;        // (clamped: channels behind dv are dropped)
#pragma unroll
    for (int kb = 0; kb < KB; ++kb) {
      const int e = kb * 16 + 8 * half;
      const bool in = e + 8 <= dk;
      o[vb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(in ? rld8(st_hi + at + e) : rz8(), qreg[kb], o[vb], 0, 0, 0);
      o[vb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(in ? rld8(st_lo + at + e) : rz8(), qreg[kb], o[vb], 0, 0, 0);
    }
  }
  {
    const float f = exp2f((float)(i + 1) * lg);
#pragma unroll
    for (int vb = 0; vb < VB; ++vb)
#pragma unroll
      for (int r = 0; r < 16; ++r) o[vb][r] *= f;
  }
  const int j_end = min(q0 + RR_BM, ch.rows);
  for (int j0 = 0; j0 < j_end; j0 += RR_BN) {
    __syncthreads();                                   // the tile before has been worked on
#pragma unroll
    for (int e0 = 0; e0 < RR_BN * CH; e0 += 256) {
      const int e = e0 + tid, r = e / CH, col = (e % CH) * 8;
      if (e < RR_BN * CH)
        *reinterpret_cast<bf16x8*>(&Ks[r * KLD + col]) =
            (col + 8 <= dk && j0 + r < ch.rows) ? rld8(k + ((size_t)(ch.row0 + j0 + r) * H + h) * dk + col) : rz8();
    }
#pragma unroll
    for (int e0 = 0; e0 < DV * 8; e0 += 256) {
      const int e = e0 + tid, d = e / 8, kc = (e % 8) * 8;
      // (columns of a tile that holds a row of the chunk were all written, zeros behind the last row)
      const bf16x8 v = d < dv ? rld8(vt + (head * dv + d) * RC + j0 + kc) : rz8();
      bf16x4 lo4, hi4;
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        lo4[x] = v[x];
        hi4[x] = v[4 + x];
      }
      *reinterpret_cast<bf16x4*>(&Vt[d * RR_VLD + kc]) = lo4;
      *reinterpret_cast<bf16x4*>(&Vt[d * RR_VLD + kc + 4]) = hi4;
    }
    __syncthreads();
    if (j0 > wi_hi || wi_lo >= ch.rows) continue;      // no row of this wave sees a key of this tile
#pragma unroll
    for (int nb = 0; nb < 2; ++nb) {                   // 32 keys at a time
      if (j0 + nb * 32 > wi_hi) break;
      f32x16 s;
#pragma unroll
      for (int r = 0; r < 16; ++r) s[r] = 0.f;
#pragma unroll
      for (int kb = 0; kb < KB; ++kb)
        s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8*>(&Ks[(nb * 32 + l32) * KLD + kb * 16 + 8 * half]),
                                                    qreg[kb], s, 0, 0, 0);
      // s[r]: key j0 + 32 nb + 8 (r/4) + 4 half + r%4 against this lane's row
      bf16x8 p_hi[2], p_lo[2];
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int d = i - (j0 + nb * 32 + 8 * (r / 4) + 4 * half + (r % 4));
        const float w = d >= 0 ? s[r] * __builtin_amdgcn_exp2f((float)d * lg) : 0.f;
        const bf16 hi = (bf16)w;
        p_hi[r / 8][r % 8] = hi;
        p_lo[r / 8][r % 8] = (bf16)(w - (float)hi);
      }
#pragma unroll
      for (int mm = 0; mm < 2; ++mm)
#pragma unroll
        for (int vb = 0; vb < VB; ++vb) {
          const bf16* vrow = &Vt[(vb * 32 + l32) * RR_VLD + nb * 32 + 16 * mm + 4 * half];
          const bf16x4 lo4 = rld4(vrow), hi4 = rld4(vrow + 8);
          bf16x8 a;
#pragma unroll
          for (int x = 0; x < 4; ++x) {
            a[x] = lo4[x];
            a[4 + x] = hi4[x];
          }
          o[vb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, p_hi[mm], o[vb], 0, 0, 0);
          o[vb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, p_lo[mm], o[vb], 0, 0, 0);
        }
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int vb = 0; vb < VB; ++vb)
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int d = vb * 32 + 8 * (r / 4) + 4 * half + (r % 4);
      if (d < dv) ss += o[vb][r] * o[vb][r];
    }
  ss += __shfl_xor(ss, 32, WAVE);
  if (!ok) return;
  const float f = 1.0f / sqrtf(ss / (float)dv + eps);
  const float* gr = gate + (size_t)row * gate_stride + (size_t)h * dv;
  bf16* op = out + ((size_t)row * H + h) * dv;
#pragma unroll
  for (int vb = 0; vb < VB; ++vb)
#pragma unroll
    for (int g4 = 0; g4 < 4; ++g4) {                   // four channels in a row (dv is a multiple of 4)
      const int d = vb * 32 + 8 * g4 + 4 * half;
      if (d >= dv) continue;
      const f32x4 g = *reinterpret_cast<const f32x4*>(gr + d);
      bf16x4 res;
#pragma unroll
      for (int x = 0; x < 4; ++x) res[x] = (bf16)(o[vb][4 * g4 + x] * f * (g[x] / (1.0f + __expf(-g[x]))));
      *reinterpret_cast<bf16x4*>(op + d) = res;
    }
}

template <int DK, int DV>
static int launch_rows(const bf16* q, const bf16* k, const bf16* vt, const bf16* st_hi, const bf16* st_lo, const float* gate,
                       int gate_stride, int H, int dk, int dv, const float* log2_decay, float eps, const int* cu, int B, int chunks,
                       bf16* out, hipStream_t st) {
  const size_t smem = ((size_t)RR_BN * (DK + 8) + (size_t)DV * RR_VLD) * sizeof(bf16);
  static bool raised = false;
  if (!raised) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&retention_rows_kernel<DK, DV>),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
    if (e != hipSuccess) {
      set_error("retention_rows: cannot have %zu bytes of LDS: %s", smem, hipGetErrorString(e));
      return 2;
    }
    raised = true;
  }
  retention_rows_kernel<DK, DV><<<dim3(2 * chunks, H), 256, smem, st>>>(q, k, vt, st_hi, st_lo, gate, gate_stride, H, dk, dv, log2_decay,
                                                                        eps, cu, B, out);
  TL_LAUNCH_CHECK("retention_rows");
  return 0;
}

}  // namespace tl

using namespace tl;

extern "C" {

int tl_retention_chunk(void) { return RC; }

// proj [n, width] = [q | k | v | g ...] float; `chunks`: the step's chunks of RC rows (every sequence's rounded up).  Scratch, in
// elements: q and k n*H*dk each, kt_hi and kt_lo chunks*H*dk*RC, vt chunks*H*dv*RC, st_hi and st_lo chunks*H*dk*dv (bfloat16),
// kv chunks*H*dk*dv (float).  out bfloat16 [n, H*dv].
int tl_retention_chunks(const float* proj, int width, int H, int dk, int dv, const int* row_pos, const float* inv_freq, int rotary_dim,
                        int interleaved, float magnitude, float kscale, const float* log2_decay, float eps, float* state,
                        long long stride, const int* cu, const int* slots, int n, int B, int chunks, void* q, void* k, void* kt_hi,
                        void* kt_lo, void* vt, float* kv, void* st_hi, void* st_lo, void* out, hipStream_t st) {
  TL_REQUIRE(n > 0 && B > 0 && B <= 65535 && H > 0 && H <= 65535 && chunks > 0, "retention_chunks: bad sizes n=%d B=%d H=%d chunks=%d", n, B,
             H, chunks);
  TL_REQUIRE(dk % 8 == 0 && dk <= RC_MAX_D && dv % 4 == 0 && dv <= RC_MAX_D && dk > 0 && dv > 0,
             "retention_chunks: heads of %d and %d are not served (keys in steps of 8, values of 4, up to %d)", dk, dv, RC_MAX_D);
  TL_REQUIRE(width >= 2 * H * (dk + dv) && width % 4 == 0, "retention_chunks: a row of %d is too short, or no multiple of 4", width);
  TL_REQUIRE(rotary_dim >= 0 && rotary_dim % 2 == 0 && rotary_dim <= dk && (rotary_dim == 0 || inv_freq),
             "retention_chunks: %d rotated channels of a head of %d", rotary_dim, dk);
  TL_REQUIRE(proj && row_pos && log2_decay && state && cu && slots && q && k && kt_hi && kt_lo && vt && kv && st_hi && st_lo && out,
             "retention_chunks: a buffer is missing");
  TL_REQUIRE(((uintptr_t)proj | (uintptr_t)q | (uintptr_t)k | (uintptr_t)kt_hi | (uintptr_t)kt_lo | (uintptr_t)vt | (uintptr_t)st_hi |
              (uintptr_t)st_lo | (uintptr_t)out) % 16 == 0, "retention_chunks: a buffer off 16 bytes");
  TL_REQUIRE(stride >= (long long)H * dk * dv, "retention_chunks: a sequence's block is too small");
  const Rotation rot{inv_freq, rotary_dim, interleaved, magnitude};
  const int wide = dk > RC_TILE ? dk : RC_TILE;
  const size_t lds = (size_t)RC_TILE * (wide + 1) * sizeof(float);
  static bool raised = false;
  if (!raised) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&retention_prepare_kernel),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, RC_TILE * (RC_MAX_D + 1) * (int)sizeof(float));
    if (e != hipSuccess) {
      set_error("retention_prepare: cannot raise its LDS: %s", hipGetErrorString(e));
      return 2;
    }
    raised = true;
  }
  retention_prepare_kernel<<<dim3(chunks * (RC / RC_TILE), H), 256, lds, st>>>(proj, width, H, dk, dv, row_pos, rot, kscale, log2_decay, cu,
                                                                              B, (bf16*)q, (bf16*)k, (bf16*)kt_hi, (bf16*)kt_lo,
                                                                              (bf16*)vt);
  TL_LAUNCH_CHECK("retention_prepare");
  retention_states_kernel<<<dim3(chunks, H, ((dk + 63) / 64) * ((dv + 63) / 64)), 256, 0, st>>>((const bf16*)kt_hi, (const bf16*)kt_lo,
                                                                                               (const bf16*)vt, H, dk, dv, cu, B, kv);
  TL_LAUNCH_CHECK("retention_states");
  retention_carry_kernel<<<dim3(((dk + 31) / 32) * ((dv + 31) / 32), H, B), 256, 0, st>>>(kv, H, dk, dv, log2_decay, state, stride, cu,
                                                                                         slots, (bf16*)st_hi, (bf16*)st_lo);
  TL_LAUNCH_CHECK("retention_carry");
  const float* gate = proj + (size_t)H * (2 * dk + dv);
#define TL_RR(DK, DV)                                                                                                        \
  return launch_rows<DK, DV>((const bf16*)q, (const bf16*)k, (const bf16*)vt, (const bf16*)st_hi, (const bf16*)st_lo, gate, \
                             width, H, dk, dv, log2_decay, eps, cu, B, chunks, (bf16*)out, st)
  if (dk <= 64 && dv <= 64) TL_RR(64, 64);
  if (dk <= 64 && dv <= 128) TL_RR(64, 128);
  if (dk <= 128 && dv <= 128) TL_RR(128, 128);
  if (dk <= 128) TL_RR(128, 256);
  TL_RR(256, 256);
#undef TL_RR
}

}  // extern "C"
