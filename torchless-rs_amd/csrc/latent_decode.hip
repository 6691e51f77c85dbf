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
// A workgroup takes one sequence, 16 heads and a share of the sequence's pages (`split` of n_splits).  A page's 64 rows
// of D = R + dr channels are staged in LDS for all its heads.  Each of the four waves makes the scores of one block of 16
// rows, S^T = K Q^T (a lane owns one head); the scores meet in LDS, and every wave goes through the softmax of all 64 rows
// and adds up a quarter of the channels, O^T += C^T P^T: the weights have the operand layout of that product as they are,
// and its other operand, the rows' channels read along the rows, the LDS hands out transposed.  The next page is under way
// into registers while this one is worked on.  Partial results (max, sum, O) meet in `part`, merged by
// latent_decode_combine_kernel; with one split the result is written at once.  More heads a workgroup would stage a page
// less often, but two workgroups of 16 heads share a compute unit where one of 32 or 64 fills it: 32 heads of a latent of
// 512 over 64 x 4,096 rows take 85 us this way and 95 with 32 heads a workgroup, 128 heads over 8 x 4,096 rows 48 and 53.
constexpr int LD_PAD = 8;

__device__ __forceinline__ s16x4 read_transposed(const bf16* p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((TL_AS3 s16x4*)p);
}

// RP >= R in steps of 64, KP >= D in steps of 32; WHOLE: D == KP, a page is one run of the memory as it is staged
template <int RP, int KP, bool WHOLE>
__global__ void __launch_bounds__(256, RP == 512 && !WHOLE ? 1 : 2)
latent_decode_kernel(const bf16* __restrict__ q, const bf16* __restrict__ pages, const int* __restrict__ table,
                     int table_stride, int ring_pages, const int* __restrict__ row_pos, int H, int R, int D, int window,
                     float scale, int n_splits, float* __restrict__ part, bf16* __restrict__ out) {
  constexpr int KB = KP / 32, VB = RP / 64, LD = KP + LD_PAD;
  constexpr int ROW_CHUNKS = KP / 8, PRE = PAGE * ROW_CHUNKS / 256;      // 16-byte chunks of a staged row; of a page, per thread
  static_assert(PAGE * ROW_CHUNKS % 256 == 0, "a page in whole rounds of loads");
  extern __shared__ __attribute__((aligned(16))) unsigned char ld_smem[];
  bf16* tile = reinterpret_cast<bf16*>(ld_smem);       // [64][LD]
  f32x4* scores = reinterpret_cast<f32x4*>(ld_smem + (size_t)PAGE * LD * sizeof(bf16));      // [4 blocks][64 lanes]
  const int b = blockIdx.x, hq0 = blockIdx.y * 16, split = blockIdx.z;
  const int tid = threadIdx.x, wave = tid / 64, lane = tid % 64, li = lane % 16, kg = lane / 16;
  const int h = min(hq0 + li, H - 1);
  const int p = row_pos[b];
  const int lo = (window > 0 && p - window + 1 > 0) ? p - window + 1 : 0;
  const int pg_lo = lo / PAGE, n_pg = p / PAGE - pg_lo + 1;
  const int my_lo = pg_lo + (int)((long long)split * n_pg / n_splits);
  const int my_hi = pg_lo + (int)((long long)(split + 1) * n_pg / n_splits);
  const int row_chunks = D / 8;

  // page pg -> registers -> LDS: channels behind D and rows behind the query's own become zeros (a row that was never
  // written may hold anything; its memory is the page's all the same)
  auto source = [&](int pg) { return pages + (size_t)table[(size_t)b * table_stride + pg % ring_pages] * PAGE * D; };
  auto chunk = [&](const bf16* src, int i) {
    if constexpr (WHOLE) return ldv8(src + (unsigned)(tid * 8) + i * 2048);
    const int c = i * 256 + tid, row = c / ROW_CHUNKS, col = c % ROW_CHUNKS;
    return col < row_chunks ? ldv8(src + (size_t)row * D + col * 8) : zv8();
  };
  auto put = [&](int i, bf16x8 v, int r1) {
    int c = i * 256 + tid;
    if constexpr (WHOLE) asm volatile("" : "+v"(c));       // (worked out for every page, not kept in registers)
    const int row = c / ROW_CHUNKS, col = c % ROW_CHUNKS;
    *reinterpret_cast<bf16x8*>(tile + row * LD + col * 8) = row <= r1 ? v : zv8();
  };
  bf16x8 ahead[PRE];
  if (my_lo < my_hi) {
    const bf16* src = source(my_lo);
#pragma unroll
    for (int i = 0; i < PRE; ++i) ahead[i] = chunk(src, i);
  }
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

  for (int pg = my_lo; pg < my_hi; ++pg) {
    const int r1 = min(p - pg * PAGE, PAGE - 1);       // the last row of the page that the query sees
    __syncthreads();                                   // the page before has been worked on
#pragma unroll
    for (int i = 0; i < PRE; ++i) put(i, ahead[i], r1);
    __syncthreads();
    if (pg + 1 < my_hi) {
      const bf16* src = source(pg + 1);
#pragma unroll
      for (int i = 0; i < PRE; ++i) ahead[i] = chunk(src, i);
    }
    {
      const bf16* krow = tile + (wave * 16 + li) * LD + 8 * kg;
      f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kb = 0; kb < KB; ++kb)
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(krow + kb * 32), qreg[kb], acc, 0, 0, 0);
      // acc[r]: row 16 wave + 4 kg + r of the page, this lane's head
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = pg * PAGE + wave * 16 + 4 * kg + r;
        acc[r] = (j <= p && j >= lo) ? acc[r] * scale : -INFINITY;
      }
      scores[wave * 64 + lane] = acc;
    }
    __syncthreads();
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
    const float alpha = __expf(m - m_new);
    float psum = 0.f;
    bf16x8 pf[2];                                      // rows 4 kg + {0..3} of blocks 2 np and 2 np + 1
#pragma unroll
    for (int blk = 0; blk < 4; ++blk)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float pv = __expf(s[blk][r] - m_new);
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
      const bf16* v0 = tile + (np * 32 + 4 * kg + li / 4) * LD + wave * VB * 16 + 4 * (li % 4);
      const bf16* v1 = v0 + 16 * LD;
#pragma unroll
      for (int vb = 0; vb < VB; ++vb) {
        typedef short s16x8 __attribute__((ext_vector_type(8)));
        const s16x4 a0 = read_transposed(v0 + vb * 16), a1 = read_transposed(v1 + vb * 16);
        const s16x8 a = __builtin_shufflevector(a0, a1, 0, 1, 2, 3, 4, 5, 6, 7);
        o[vb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), pf[np], o[vb], 0, 0, 0);
      }
    }
  }
  // o[vb][r] = O[channel 16 (wave VB + vb) + 4 kg + r][head li]; m and l are the same in all waves
  if (hq0 + li >= H) return;
  const size_t bh = (size_t)b * H + hq0 + li;
  float* dst = part + (bh * n_splits + split) * (size_t)(R + 2);
  const float inv = 1.0f / l;
#pragma unroll
  for (int vb = 0; vb < VB; ++vb)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int c = 16 * (wave * VB + vb) + 4 * kg + r;
      if (c >= R) continue;
      if (n_splits == 1) out[bh * R + c] = (bf16)(o[vb][r] * inv);
      else dst[2 + c] = o[vb][r];
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
  const size_t bh = blockIdx.x, line = (size_t)R + 2;
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
      const float f = ms == -INFINITY ? 0.f : __expf(ms - mm);
      f_s[t] = f;
      w = f * p[(s0 + t) * line + 1];
    }
    ll += block_sum<256>(w, sh);
    __syncthreads();
    if (c < R) {
      const float* v = p + s0 * line + 2 + c;
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

template <int RP, int KP, bool WHOLE>
static int launch_latent_decode_v(const bf16* q, const bf16* pages, const int* table, int table_stride, int ring_pages,
                                const int* row_pos, int B, int H, int R, int D, int window, float scale, int n_splits, float* part,
                                bf16* out, hipStream_t st) {
  const size_t smem = (size_t)PAGE * (KP + LD_PAD) * sizeof(bf16) + 4 * 64 * sizeof(f32x4);
  static bool raised = false;
  if (!raised) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_decode_kernel<RP, KP, WHOLE>),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
    if (e != hipSuccess) {
      set_error("latent_decode: cannot have %zu bytes of LDS: %s", smem, hipGetErrorString(e));
      return 2;
    }
    raised = true;
  }
  const dim3 grid(B, (H + 15) / 16, n_splits);
  latent_decode_kernel<RP, KP, WHOLE><<<grid, 256, smem, st>>>(q, pages, table, table_stride, ring_pages, row_pos, H, R, D, window, scale,
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
                                const int* row_pos, int B, int H, int R, int D, int window, float scale, int n_splits, float* part,
                                bf16* out, hipStream_t st) {
  if (D == KP)
    return launch_latent_decode_v<RP, KP, true>(q, pages, table, table_stride, ring_pages, row_pos, B, H, R, D, window, scale,
                                                    n_splits, part, out, st);
  return launch_latent_decode_v<RP, KP, false>(q, pages, table, table_stride, ring_pages, row_pos, B, H, R, D, window, scale,
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

// q [B, H, D], pages rows of D = R + dr channels, part: B * H * n_splits * (R + 2) floats (n_splits > 1)
int tl_latent_decode_bf16(const void* q, const void* pages, const int* table, int table_stride, int ring_pages, const int* row_pos,
                          int B, int H, int R, int dr, int window, float scale, int n_splits, float* part, void* out,
                          hipStream_t st) {
  const int D = R + dr;
  TL_REQUIRE(B >= 0 && H > 0 && R > 0 && dr >= 0 && R <= 512 && D <= 576 && D % 8 == 0 && window >= 0,
             "latent_decode: bad sizes B=%d H=%d R=%d dr=%d window=%d (latents up to 512, rows up to 576 in steps of 8)", B, H, R, dr,
             window);
  TL_REQUIRE(q && pages && table && row_pos && out && table_stride > 0 && ring_pages > 0, "latent_decode: a buffer is missing");
  TL_REQUIRE((uintptr_t)q % 16 == 0 && (uintptr_t)pages % 16 == 0, "latent_decode: queries and pages must be 16-byte aligned");
  TL_REQUIRE(n_splits >= 1 && n_splits <= 65535 && (n_splits == 1 || part), "latent_decode: %d splits need room for their sums", n_splits);
  if (B == 0) return 0;
#define TL_LD(RP, KP)                                                                                                              \
  return launch_latent_decode<RP, KP>((const bf16*)q, (const bf16*)pages, table, table_stride, ring_pages, row_pos, B, H, R, D,    \
                                      window, scale, n_splits, part, (bf16*)out, st)
  if (R <= 64 && D <= 96) TL_LD(64, 96);
  if (R <= 128 && D <= 192) TL_LD(128, 192);
  if (R <= 256 && D <= 288) TL_LD(256, 288);
  if (R <= 256 && D <= 320) TL_LD(256, 320);
  TL_LD(512, 576);
#undef TL_LD
}

}  // extern "C"
