// Single tokens over cached latents on the matrix cores (see latent_cache.hip for the mechanism): the
// products per head that lead into the latent's channels and out of them, and the attention over the
// cached rows, which are keys and values of all heads at once.
#include "common.hpp"

namespace tl {

#define TL_AS3 __attribute__((address_space(3)))
typedef short s16x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ bf16x8 ldv8(const bf16* p) { return *reinterpret_cast<const bf16x8*>(p); }
__device__ __forceinline__ bf16x8 zv8() {
  bf16x8 z;
#pragma unroll
  for (int i = 0; i < 8; ++i) z[i] = (bf16)0.f;
  return z;
}

// ---- products per head ----------------------------------------------------------------------------------
// out[n, h, j] = sum_k w[h, j, k] x[n, h, k] for 16 rows n at a time.  SPLIT: a workgroup owns 16 outputs and its
// four waves share K; else it owns 64, 16 a wave.
template <bool SPLIT>
__global__ void __launch_bounds__(256)
head_products_mfma_kernel(const bf16* __restrict__ x, const bf16* __restrict__ w, int n_rows, int H, int N, int K,
                          bf16* __restrict__ out, long long out_row, long long out_head) {
  __shared__ f32x4 red[SPLIT ? 4 : 1][64];
  const int h = blockIdx.y, n0 = blockIdx.z * 16;
  const int wave = threadIdx.x / 64, lane = threadIdx.x % 64, li = lane % 16, kg = lane / 16;
  const int j0 = SPLIT ? blockIdx.x * 16 : blockIdx.x * 64 + wave * 16;
  const bf16* wr = w + ((size_t)h * N + min(j0 + li, N - 1)) * K;            // (clamped: sums of lanes without an output are dropped)
  const bf16* xr = x + ((size_t)min(n0 + li, n_rows - 1) * H + h) * K;
  f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
  const int steps = (K + 31) / 32;
  const int per = SPLIT ? (steps + 3) / 4 : steps;
  const int s0 = SPLIT ? wave * per : 0, s1 = min(steps, s0 + per);
#pragma unroll 4
  for (int s = s0; s < s1; ++s) {
    const int k = s * 32 + 8 * kg;
    const bool ok = k + 8 <= K;
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ok ? ldv8(wr + k) : zv8(), ok ? ldv8(xr + k) : zv8(), acc, 0, 0, 0);
  }
  if constexpr (SPLIT) {
    red[wave][lane] = acc;
    __syncthreads();
    if (wave != 0) return;
    acc = (red[0][lane] + red[1][lane]) + (red[2][lane] + red[3][lane]);
  }
  if (n0 + li >= n_rows) return;
  bf16* o = out + (size_t)(n0 + li) * out_row + (size_t)h * out_head + j0 + 4 * kg;
#pragma unroll
  for (int r = 0; r < 4; ++r)
    if (j0 + 4 * kg + r < N) o[r] = (bf16)acc[r];
}

// ---- attention ------------------------------------------------------------------------------------------
// A workgroup takes one sequence, HB blocks of 16 heads and a share of the sequence's pages (`split` of n_splits).  A page's
// 64 rows of D = R + dr channels are staged in LDS for all its heads.  Each of a head block's four waves makes the scores of
// one block of 16 rows, S^T = K Q^T (a lane owns one head); the scores meet in LDS, and every wave goes through the softmax
// of all 64 rows and adds up a quarter of the channels, O^T += C^T P^T: the weights have the operand layout of that product
// as they are, and its other operand, the rows' channels read along the rows, the LDS hands out transposed.  The next page
// is under way into registers while this one is worked on; with HB == 2 it is staged beside this one, too.  Partial results
// (max, sum, O; the maximum as an exponent of 2) meet in `part`, merged by latent_decode_combine_kernel; with one split the
// result is written at once.  HB == 1: two workgroups share a compute unit; HB == 2 (one fills it): a page is fetched half
// as often, which pays as soon as every unit has more than a few pages to go through (32 heads of a latent of 512: 64 x
// 4,096 rows take 73 us against 82, 8 x 4,096 rows 25 against 22).
// A staged row takes an odd multiple of 64 channels and keeps its 16-byte chunks in another order within each eight, by
// row: then none of the accesses meets itself in a bank (the rows of a page as they are written, 16 rows of 8 channels for
// the scores, 8 rows of 16 channels read transposed).
constexpr int staged_row(int channels) { return (channels + 63) / 64 % 2 ? (channels + 63) / 64 * 64 : (channels + 127) / 64 * 64; }
__device__ __forceinline__ int chunk_order(int row) { return ((row >> 1) & 3) << 1 | ((row >> 3) & 1); }

__device__ __forceinline__ s16x4 read_transposed(const bf16* p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((TL_AS3 s16x4*)p);
}

// one split's result: [max, sum, -, - | O]
__host__ __device__ __forceinline__ int part_line(int R) { return 4 + (R + 3) / 4 * 4; }

// RP >= R in steps of 64, KP >= D in steps of 32; WHOLE: D == KP, a page is one run of the memory as it is staged
template <int RP, int KP, int HB, bool WHOLE>
__global__ void __launch_bounds__(256 * HB, (RP == 512 && !WHOLE) || HB == 2 ? 1 : 2)
latent_decode_kernel(const bf16* __restrict__ q, const bf16* __restrict__ pages, const int* __restrict__ table,
                     int table_stride, int ring_pages, const int* __restrict__ row_pos, int H, int R, int D, int window,
                     float scale, int n_splits, float* __restrict__ part, bf16* __restrict__ out) {
  constexpr int KB = KP / 32, VB = RP / 64, LD = staged_row(KP), CB = (KP + 63) / 64, HALVES = 2 / HB, BUFS = HB;
  extern __shared__ __attribute__((aligned(16))) unsigned char ld_smem[];
  bf16* tile = reinterpret_cast<bf16*>(ld_smem);       // [BUFS][64][LD]
  f32x4* scores = reinterpret_cast<f32x4*>(ld_smem + (size_t)BUFS * PAGE * LD * sizeof(bf16)) + (threadIdx.x / 256) * 256;      // [HB][4 blocks][64 lanes]
  const int b = blockIdx.x, hq0 = (blockIdx.y * HB + threadIdx.x / 256) * 16, split = blockIdx.z;
  const int tid = threadIdx.x, wave = tid / 64 % 4, lane = tid % 64, li = lane % 16, kg = lane / 16;
  const int h = min(hq0 + li, H - 1);
  const int p = row_pos[b];
  const int lo = (window > 0 && p - window + 1 > 0) ? p - window + 1 : 0;
  const int pg_lo = lo / PAGE, n_pg = p / PAGE - pg_lo + 1;
  const int my_lo = pg_lo + (int)((long long)split * n_pg / n_splits);
  const int my_hi = pg_lo + (int)((long long)(split + 1) * n_pg / n_splits);

  // page pg -> registers -> LDS: eight lanes a row and 64 channels at a time (HB == 1: rows row and row + 32 of the page)
  const int row = tid / 8, col = tid % 8;
  bf16x8 ahead[HALVES][CB];
  auto load = [&](int pg) {
    const bf16* src = pages + (size_t)table[(size_t)b * table_stride + pg % ring_pages] * PAGE * D + (unsigned)(row * D + col * 8);
#pragma unroll
    for (int half = 0; half < HALVES; ++half)
#pragma unroll
      for (int i = 0; i < CB; ++i)                     // (channels behind D become zeros)
        ahead[half][i] = ((WHOLE && KP % 64 == 0) || i * 64 + col * 8 < D) ? ldv8(src + (unsigned)(half * 32 * D + i * 64)) : zv8();
  };
  bf16* const put_at = tile + row * LD + (col ^ chunk_order(row)) * 8;      // (row + 32 has the same order)
  auto put = [&](int pg, int at) {
    const int r1 = p - pg * PAGE;                      // the last row of the page that the query sees, if it is in the page
#pragma unroll
    for (int half = 0; half < HALVES; ++half) {
      // rows behind the query's own become zeros: one that was never written may hold anything
      if (r1 < PAGE - 1 && row + half * 32 > r1) {
#pragma unroll
        for (int i = 0; i < CB; ++i) ahead[half][i] = zv8();
      }
#pragma unroll
      for (int i = 0; i < CB; ++i) *reinterpret_cast<bf16x8*>(put_at + at + half * 32 * LD + i * 64) = ahead[half][i];
    }
  };
  if (my_lo < my_hi) load(my_lo);
  bf16x8 qreg[KB];
  {
    const bf16* qp = q + ((size_t)b * H + h) * D;
#pragma unroll
    for (int kb = 0; kb < KB; ++kb) {
      const int k = kb * 32 + 8 * kg;
      qreg[kb] = (k + 8 <= D) ? ldv8(qp + k) : zv8();
    }
  }
  f32x4 o[VB];
#pragma unroll
  for (int vb = 0; vb < VB; ++vb) o[vb] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;

  if constexpr (BUFS == 2) {
    if (my_lo < my_hi) put(my_lo, 0);
    if (my_lo + 1 < my_hi) load(my_lo + 1);
  }
  const float scale2 = scale * 1.44269504f;
  const int sw = chunk_order(li);
  for (int pg = my_lo; pg < my_hi; ++pg) {
    const int r1 = p - pg * PAGE;                      // the last row of the page that the query sees, if it is in the page
    const bool whole = r1 >= PAGE - 1 && pg * PAGE >= lo;
    if constexpr (BUFS == 1) {
      __syncthreads();                                 // the page before has been worked on
      put(pg, 0);
    }
    __syncthreads();
    if constexpr (BUFS == 1) {
      if (pg + 1 < my_hi) load(pg + 1);
    }
    const int at = BUFS == 1 ? 0 : (pg - my_lo) % 2 * PAGE * LD;
    {
      const bf16* krow = tile + at + (wave * 16 + li) * LD;
      f32x4 two[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};      // two chains: one does not wait for the other
      const bf16* kc[2] = {krow + (kg ^ sw) * 8, krow + ((4 + kg) ^ sw) * 8};
#pragma unroll
      for (int kb = 0; kb < KB; ++kb)
        two[kb % 2] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(kc[kb % 2] + kb / 2 * 64), qreg[kb],
                                                              two[kb % 2], 0, 0, 0);
      f32x4 acc = two[0] + two[1];
      // acc[r]: row 16 wave + 4 kg + r of the page, this lane's head
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[r] *= scale2;
      if (!whole) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = pg * PAGE + wave * 16 + 4 * kg + r;
          if (j > p || j < lo) acc[r] = -INFINITY;
        }
      }
      scores[wave * 64 + lane] = acc;
    }
    __syncthreads();
    if constexpr (BUFS == 2) {
      if (pg + 1 < my_hi) put(pg + 1, PAGE * LD - at);
      if (pg + 2 < my_hi) load(pg + 2);
    }
    f32x4 s[4];
#pragma unroll
    for (int blk = 0; blk < 4; ++blk) s[blk] = scores[blk * 64 + lane];
    float tmax = -INFINITY;
#pragma unroll
    for (int blk = 0; blk < 4; ++blk)
#pragma unroll
      for (int r = 0; r < 4; ++r) tmax = fmaxf(tmax, s[blk][r]);
    tmax = fmaxf(tmax, __shfl_xor(tmax, 16, WAVE));
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, WAVE));
    const float m_new = fmaxf(m, tmax);                // finite: the page holds a visible row
    const float alpha = __builtin_amdgcn_exp2f(m - m_new);
    float psum = 0.f;
    bf16x8 pf[2];                                      // rows 4 kg + {0..3} of blocks 2 np and 2 np + 1
#pragma unroll
    for (int blk = 0; blk < 4; ++blk)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float pv = __builtin_amdgcn_exp2f(s[blk][r] - m_new);
        psum += pv;
        pf[blk / 2][4 * (blk % 2) + r] = (bf16)pv;
      }
    psum += __shfl_xor(psum, 16, WAVE);
    psum += __shfl_xor(psum, 32, WAVE);
    l = l * alpha + psum;
    m = m_new;
    if (__ballot(alpha != 1.0f) != 0ull) {             // the running maximum moved in some lane
#pragma unroll
      for (int vb = 0; vb < VB; ++vb)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[vb][r] *= alpha;
    }
    // lane (kg, li) names rows 4 kg + li / 4 and channels 4 (li % 4) .. + 3 of a block and receives channel li of rows
    // 4 kg .. + 3
#pragma unroll
    for (int np = 0; np < 2; ++np) {
      const bf16* vrow = tile + at + (np * 32 + 4 * kg + li / 4) * LD + (li % 2) * 4;
#pragma unroll
      for (int vb = 0; vb < VB; ++vb) {
        typedef short s16x8 __attribute__((ext_vector_type(8)));
        const int ch = (wave * VB + vb) * 2 + (li % 4) / 2;                       // the chunk that this lane names
        const bf16* v0 = vrow + (ch ^ chunk_order(4 * kg + li / 4)) * 8;
        const s16x4 a0 = read_transposed(v0), a1 = read_transposed(v0 + 16 * LD);
        const s16x8 a = __builtin_shufflevector(a0, a1, 0, 1, 2, 3, 4, 5, 6, 7);
        o[vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), pf[np], o[vb], 0, 0, 0);
      }
    }
  }
  // o[vb][r] = O[channel 16 (wave VB + vb) + 4 kg + r][head li]; m and l are the same in all waves of a head
  if (hq0 + li >= H) return;
  const size_t bh = (size_t)b * H + hq0 + li;
  float* dst = part + (bh * n_splits + split) * (size_t)part_line(R);
  const float inv = 1.0f / l;
#pragma unroll
  for (int vb = 0; vb < VB; ++vb) {
    const int c = 16 * (wave * VB + vb) + 4 * kg;
    if (n_splits > 1) {                                // (a line's end is padded to whole fours)
      if (c < R) *reinterpret_cast<f32x4*>(dst + 4 + c) = o[vb];
      continue;
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) o[vb][r] *= inv;
    if (c + 4 <= R && R % 4 == 0) {
      bf16x4 v;
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = (bf16)o[vb][r];
      *reinterpret_cast<bf16x4*>(out + bh * R + c) = v;
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (c + r < R) out[bh * R + c + r] = (bf16)o[vb][r];
    }
  }
  if (n_splits > 1 && wave == 0 && kg == 0) {
    dst[0] = m;
    dst[1] = l;
  }
}

// The splits of a (sequence, head) become its row of the result: 256 channels a workgroup.
constexpr int LD_MERGE = 256;          // splits whose factors are worked out at a time

__global__ void __launch_bounds__(256)
latent_decode_combine_kernel(const float* __restrict__ part, int n_splits, int R, bf16* __restrict__ out) {
  __shared__ float f_s[LD_MERGE];
  __shared__ float sh[4];
  const size_t bh = blockIdx.x, line = part_line(R);
  const float* p = part + bh * n_splits * line;
  const int t = threadIdx.x, c = blockIdx.y * 256 + t;
  float mm = -INFINITY;
  for (int s = t; s < n_splits; s += 256) mm = fmaxf(mm, p[s * line]);
  mm = block_max<256>(mm, sh);
  float ll = 0.f, acc = 0.f;
  for (int s0 = 0; s0 < n_splits; s0 += LD_MERGE) {
    const int n = min(LD_MERGE, n_splits - s0);
    __syncthreads();
    float w = 0.f;
    if (t < n) {
      const float ms = p[(s0 + t) * line];
      const float f = ms == -INFINITY ? 0.f : exp2f(ms - mm);
      f_s[t] = f;
      w = f * p[(s0 + t) * line + 1];
    }
    ll += block_sum<256>(w, sh);
    __syncthreads();
    if (c < R) {
      const float* v = p + s0 * line + 4 + c;
      int s = 0;
      for (; s + 8 <= n; s += 8) {
        float x[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) x[i] = v[(s + i) * line];
#pragma unroll
        for (int i = 0; i < 8; ++i) acc = fmaf(x[i], f_s[s + i], acc);
      }
      for (; s < n; ++s) acc = fmaf(v[s * line], f_s[s], acc);
    }
  }
  if (c < R) out[bh * R + c] = (bf16)(acc / ll);
}

template <int RP, int KP, int HB, bool WHOLE>
static int launch_latent_decode_v(const bf16* q, const bf16* pages, const int* table, int table_stride, int ring_pages,
                                const int* row_pos, int B, int H, int R, int D, int window, float scale, int n_splits, float* part,
                                bf16* out, hipStream_t st) {
  const size_t smem = HB * ((size_t)PAGE * staged_row(KP) * sizeof(bf16) + 4 * 64 * sizeof(f32x4));
  static bool raised = false;
  if (!raised) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_decode_kernel<RP, KP, HB, WHOLE>),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
    if (e != hipSuccess) {
      set_error("latent_decode: cannot have %zu bytes of LDS: %s", smem, hipGetErrorString(e));
      return 2;
    }
    raised = true;
  }
  const dim3 grid(B, (H + 16 * HB - 1) / (16 * HB), n_splits);
  latent_decode_kernel<RP, KP, HB, WHOLE><<<grid, 256 * HB, smem, st>>>(q, pages, table, table_stride, ring_pages, row_pos, H, R, D, window, scale,
                                                            n_splits, part, out);
  TL_LAUNCH_CHECK("latent_decode");
  if (n_splits > 1) {
    latent_decode_combine_kernel<<<dim3(B * H, (R + 255) / 256), 256, 0, st>>>(part, n_splits, R, out);
    TL_LAUNCH_CHECK("latent_decode_combine");
  }
  return 0;
}

template <int RP, int KP>
static int launch_latent_decode(const bf16* q, const bf16* pages, const int* table, int table_stride, int ring_pages,
                                const int* row_pos, int B, int H, int R, int D, int window, float scale, int n_splits,
                                int head_blocks, float* part, bf16* out, hipStream_t st) {
  if constexpr (KP == 576) {
    if (head_blocks == 2 && D == KP)
      return launch_latent_decode_v<RP, KP, 2, true>(q, pages, table, table_stride, ring_pages, row_pos, B, H, R, D, window, scale,
                                                     n_splits, part, out, st);
  }
  if (D == KP)
    return launch_latent_decode_v<RP, KP, 1, true>(q, pages, table, table_stride, ring_pages, row_pos, B, H, R, D, window, scale,
                                                    n_splits, part, out, st);
  return launch_latent_decode_v<RP, KP, 1, false>(q, pages, table, table_stride, ring_pages, row_pos, B, H, R, D, window, scale,
                                                   n_splits, part, out, st);
}

}  // namespace tl

using namespace tl;

extern "C" {

// bfloat16, K % 8 == 0
int tl_head_products_bf16(const void* x, const void* w, int n, int H, int N, int K, void* out, long long out_row, long long out_head,
                          int units, hipStream_t st) {
  TL_REQUIRE(n >= 0 && n <= 1 << 20 && H > 0 && H <= 65535 && N > 0 && K > 0 && K % 8 == 0 && out_head >= N,
             "head_products: bad sizes n=%d H=%d N=%d K=%d", n, H, N, K);
  TL_REQUIRE(x && w && out && (uintptr_t)x % 16 == 0 && (uintptr_t)w % 16 == 0, "head_products: a buffer is missing or off 16 bytes");
  if (n == 0) return 0;
  const int rows = (n + 15) / 16;
  if ((long long)((N + 63) / 64) * H * rows < 2 * units && K >= 128)
    head_products_mfma_kernel<true><<<dim3((N + 15) / 16, H, rows), 256, 0, st>>>((const bf16*)x, (const bf16*)w, n, H, N, K,
                                                                                  (bf16*)out, out_row, out_head);
  else
    head_products_mfma_kernel<false><<<dim3((N + 63) / 64, H, rows), 256, 0, st>>>((const bf16*)x, (const bf16*)w, n, H, N, K,
                                                                                   (bf16*)out, out_row, out_head);
  TL_LAUNCH_CHECK("head_products_mfma");
  return 0;
}

// q [B, H, D], pages rows of D = R + dr channels, head_blocks: of 16 heads a workgroup (2: rows of 576 channels, else 1 is
// taken), part: tl_latent_part_line(R) floats for each of B * H * n_splits (n_splits > 1)
int tl_latent_part_line(int R) { return part_line(R); }

int tl_latent_decode_bf16(const void* q, const void* pages, const int* table, int table_stride, int ring_pages, const int* row_pos,
                          int B, int H, int R, int dr, int window, float scale, int n_splits, int head_blocks, float* part,
                          void* out, hipStream_t st) {
  const int D = R + dr;
  TL_REQUIRE(B >= 0 && H > 0 && R > 0 && dr >= 0 && R <= 512 && D <= 576 && D % 8 == 0 && window >= 0,
             "latent_decode: bad sizes B=%d H=%d R=%d dr=%d window=%d (latents up to 512, rows up to 576 in steps of 8)", B, H, R, dr,
             window);
  TL_REQUIRE(q && pages && table && row_pos && out && table_stride > 0 && ring_pages > 0, "latent_decode: a buffer is missing");
  TL_REQUIRE((uintptr_t)q % 16 == 0 && (uintptr_t)pages % 16 == 0, "latent_decode: queries and pages must be 16-byte aligned");
  TL_REQUIRE(n_splits >= 1 && n_splits <= 65535 && (n_splits == 1 || part), "latent_decode: %d splits need room for their sums", n_splits);
  TL_REQUIRE((head_blocks == 1 || head_blocks == 2) && (uintptr_t)part % 16 == 0 && (uintptr_t)out % 8 == 0,
             "latent_decode: %d blocks of heads, or a result off its alignment", head_blocks);
  if (B == 0) return 0;
#define TL_LD(RP, KP)                                                                                                              \
  return launch_latent_decode<RP, KP>((const bf16*)q, (const bf16*)pages, table, table_stride, ring_pages, row_pos, B, H, R, D,    \
                                      window, scale, n_splits, head_blocks, part, (bf16*)out, st)
  if (R <= 64 && D <= 96) TL_LD(64, 96);
  if (R <= 128 && D <= 192) TL_LD(128, 192);
  if (R <= 256 && D <= 288) TL_LD(256, 288);
  if (R <= 256 && D <= 320) TL_LD(256, 320);
  TL_LD(512, 576);
#undef TL_LD
}

}  // extern "C"
