// Attention whose cache keeps, per position, a latent and one rotated key part that all heads share:
// row [c (R) | k_r (dr)] of a page [64][R + dr], nothing per head.
//
//   q_h = [q_n (dn) | q_r (dr)] of W_q h ,  q_r rotated by position
//   c = rms(a) * w ,  k_r = b rotated       with [a | b] = W_dkv h
//   k_h = [W_uk[h] c | k_r] ,  v_h = W_uv[h] c
//   score = (q_n . W_uk[h] c + q_r . k_r) * scale ,  out_h = sum of softmax weights * v_h
//
// Steps with several rows a sequence make k_h and v_h of the step's rows, and of the cached
// positions they look back to (`latent_gather`, a product, `latent_heads` into pages of the usual
// kind that live for the step alone), and run the attention of keys and values per head.  Steps of
// single tokens never make them: q_n goes through W_uk[h]^T to the latent's channels
// (`head_products`), the attention runs over the cached rows as they are, all heads over the same
// ones, and its sums over c go through W_uv[h].
#include "common.hpp"

namespace tl {

constexpr int LC_MAX_R = 1024;        // most channels of a latent
constexpr int LC_MAX_ROT = 256;       // most rotated channels

// Where the four pieces of a row go.  q_n and q_r: base + n * row + head * head_stride (elements).
template <typename T>
struct LatentOut {
  T* qn;
  long long qn_row, qn_head;
  T* qr;
  long long qr_row, qr_head;
  T* c;                    // [n, R] or null
  T* rows;                 // [n, R + dr] or null
  T* pages;                // or null: row n is sequence n's only one and goes to the page of its position
  const int* table;
  int table_stride, ring_pages;
};

constexpr int LP_HEADS = 8;           // heads of a workgroup

// blockIdx.y 0: the latent and the rotated key part; y > 0: LP_HEADS heads of q.
template <typename T>
__global__ void __launch_bounds__(256)
latent_prepare_kernel(const float* __restrict__ qf, int q_stride, const float* __restrict__ cf, int c_stride, int H, int dn,
                      int dr, int R, const float* __restrict__ w, float eps, const int* __restrict__ row_pos, Rotation rot,
                      LatentOut<T> out) {
  __shared__ float cs_s[LC_MAX_ROT / 2], sn_s[LC_MAX_ROT / 2], sh[4];
  const int n = blockIdx.x, t = threadIdx.x;
  const int pos = row_pos[n];
  const int half = dr / 2;             // (dr is even) pairs behind rotary_dim / 2 pass through
  for (int i = t; i < half; i += 256) {
    float sn = 0.f, cs = 1.f;
    if (2 * i < rot.rotary_dim) {
      sincosf((float)pos * rot.inv_freq[i], &sn, &cs);
      cs *= rot.magnitude;
      sn *= rot.magnitude;
    }
    cs_s[i] = cs;
    sn_s[i] = sn;
  }
  __syncthreads();
  if (blockIdx.y == 0) {
    const float* row = cf + (size_t)n * c_stride;
    float ss = 0.f;
    for (int i = t; i < R; i += 256) ss += row[i] * row[i];
    ss = block_sum<256>(ss, sh);
    const float rms = sqrtf(ss / (float)R + eps);
    T* line = out.rows ? out.rows + (size_t)n * (R + dr) : nullptr;
    if (out.pages) {
      const int page = out.table[(size_t)n * out.table_stride + (pos / PAGE) % out.ring_pages];
      line = out.pages + ((size_t)page * PAGE + pos % PAGE) * (R + dr);
    }
    for (int i = t; i < R; i += 256) {
      const T v = from_f32<T>((row[i] / rms) * w[i]);
      if (out.c) out.c[(size_t)n * R + i] = v;
      if (line) line[i] = v;
    }
    if (line)
      for (int i = t; i < half; i += 256) {
        int a, b;
        pair_channels(i, rot.rotary_dim, rot.interleaved, a, b);
        float x, y;
        rotate_pair(row[R + a], row[R + b], cs_s[i], sn_s[i], x, y);
        line[R + a] = from_f32<T>(x);
        line[R + b] = from_f32<T>(y);
      }
    return;
  }
  const int h0 = (blockIdx.y - 1) * LP_HEADS, hn = min(LP_HEADS, H - h0);
  const float* row = qf + (size_t)n * q_stride + (size_t)h0 * (dn + dr);
  T* qn = out.qn + (size_t)n * out.qn_row + (size_t)h0 * out.qn_head;
  T* qr = out.qr + (size_t)n * out.qr_row + (size_t)h0 * out.qr_head;
  for (int e = t; e < hn * dn; e += 256) {
    const int h = e / dn, i = e % dn;
    qn[h * out.qn_head + i] = from_f32<T>(row[h * (dn + dr) + i]);
  }
  for (int e = t; e < hn * half; e += 256) {
    const int h = e / half, i = e % half;
    int a, b;
    pair_channels(i, rot.rotary_dim, rot.interleaved, a, b);
    const float* p = row + h * (dn + dr) + dn;
    float x, y;
    rotate_pair(p[a], p[b], cs_s[i], sn_s[i], x, y);
    qr[h * out.qr_head + a] = from_f32<T>(x);
    qr[h * out.qr_head + b] = from_f32<T>(y);
  }
}

// rows [n, D] into the pages of their positions; a row that the same step overwrites in a ring is skipped
template <typename T>
__global__ void __launch_bounds__(256)
latent_commit_kernel(const T* __restrict__ rows, const int* __restrict__ row_seq, const int* __restrict__ row_pos,
                     const int* __restrict__ len_after, const int* __restrict__ table, int table_stride, int ring_pages, int D,
                     T* __restrict__ pages) {
  const int n = blockIdx.x, b = row_seq[n], p = row_pos[n];
  if ((long long)p < (long long)len_after[b] - (long long)ring_pages * PAGE) return;
  const int page = table[(size_t)b * table_stride + (p / PAGE) % ring_pages];
  T* line = pages + ((size_t)page * PAGE + p % PAGE) * D;
  for (int i = threadIdx.x; i < D; i += 256) line[i] = rows[(size_t)n * D + i];
}

// The cached latents of a step's sequences, page after page: page g of the result is page g - off[b] of sequence b's
// part of the table, off [B + 1] the running number of pages.  c [pages * 64, R], kr [pages * 64, dr].
template <typename T>
__global__ void __launch_bounds__(256)
latent_gather_kernel(const T* __restrict__ pages, const int* __restrict__ table, int table_stride, const int* __restrict__ off,
                     int B, int R, int dr, T* __restrict__ c, T* __restrict__ kr) {
  const int g = blockIdx.x;
  int b = 0;
  while (b < B && off[b + 1] <= g) ++b;
  if (b == B) return;
  const int page = table[(size_t)b * table_stride + g - off[b]];
  const int D = R + dr;
  const T* src = pages + (size_t)page * PAGE * D;
  for (int e = blockIdx.y * 256 + threadIdx.x; e < PAGE * D; e += gridDim.y * 256) {
    const int r = e / D, i = e % D;
    const size_t line = (size_t)g * PAGE + r;
    if (i < R) c[line * R + i] = src[e];
    else kr[line * dr + i - R] = src[e];
  }
}

// kvf float [n, H*dn + H*dv] = [keys of all heads | values of all heads], kr [n, kr_stride ...]: k [n, H, dn + dr] and
// v [n, H, dv]; a workgroup takes LH_CHUNK outputs of a row.
constexpr int LH_CHUNK = 2048;
template <typename T>
__global__ void __launch_bounds__(256)
latent_heads_kernel(const float* __restrict__ kvf, const T* __restrict__ kr, int kr_stride, int H, int dn, int dr, int dv,
                    T* __restrict__ k, T* __restrict__ v) {
  const int n = blockIdx.x, dk = dn + dr, K = H * dk, V = H * dv;
  const float* row = kvf + (size_t)n * H * (dn + dv);
  const int e1 = min(K + V, (int)(blockIdx.y + 1) * LH_CHUNK);
  for (int e = blockIdx.y * LH_CHUNK + threadIdx.x; e < e1; e += 256) {
    if (e < K) {
      const int h = e / dk, i = e % dk;
      k[(size_t)n * K + e] = i < dn ? from_f32<T>(row[h * dn + i]) : kr[(size_t)n * kr_stride + i - dn];
    } else {
      v[(size_t)n * V + e - K] = from_f32<T>(row[H * dn + e - K]);
    }
  }
}

// The same for gathered pages: page g of `out` = [keys [H][64][dn + dr] | values [H][dv][64]].
template <typename T>
__global__ void __launch_bounds__(256)
latent_heads_pages_kernel(const float* __restrict__ kvf, const T* __restrict__ kr, int H, int dn, int dr, int dv,
                          T* __restrict__ out) {
  __shared__ float tile[PAGE][PAGE + 1];
  const int g = blockIdx.x, h = blockIdx.y, dk = dn + dr, t = threadIdx.x;
  const size_t width = (size_t)H * (dn + dv);
  const float* rows = kvf + (size_t)g * PAGE * width;
  T* kd = out + (size_t)g * H * PAGE * (dk + dv) + (size_t)h * PAGE * dk;
  T* vd = out + (size_t)g * H * PAGE * (dk + dv) + (size_t)H * PAGE * dk + (size_t)h * PAGE * dv;
  for (int e = t; e < PAGE * dk; e += 256) {
    const int r = e / dk, i = e % dk;
    kd[e] = i < dn ? from_f32<T>(rows[r * width + (size_t)h * dn + i]) : kr[((size_t)g * PAGE + r) * dr + i - dn];
  }
  for (int d0 = 0; d0 < dv; d0 += PAGE) {
    const int m = min(PAGE, dv - d0);
    __syncthreads();
    for (int e = t; e < PAGE * PAGE; e += 256) {
      const int r = e / PAGE, i = e % PAGE;
      if (i < m) tile[r][i] = rows[r * width + (size_t)H * dn + (size_t)h * dv + d0 + i];
    }
    __syncthreads();
    for (int e = t; e < m * PAGE; e += 256) {
      const int i = e / PAGE, r = e % PAGE;
      vd[(size_t)(d0 + i) * PAGE + r] = from_f32<T>(tile[r][i]);
    }
  }
}

// out[n, h, j] = sum_k w[h, j, k] x[n, h, k], float sums; x [n, H, K], w [H, N, K], out: base + n * out_row + h *
// out_head + j.  One wave an output at a time.
template <typename T>
__global__ void __launch_bounds__(256)
head_products_kernel(const T* __restrict__ x, const T* __restrict__ w, int H, int N, int K, T* __restrict__ out,
                     long long out_row, long long out_head) {
  const int n = blockIdx.z, h = blockIdx.y, lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
  const T* xr = x + ((size_t)n * H + h) * K;
  for (int i = 0; i < 8; ++i) {
    const int j = blockIdx.x * 32 + wave * 8 + i;
    if (j >= N) break;
    const T* wr = w + ((size_t)h * N + j) * K;
    float acc = 0.f;
    for (int c = lane; c < K; c += WAVE) acc = fmaf(to_f32(wr[c]), to_f32(xr[c]), acc);
    acc = wave_sum(acc);
    if (lane == 0) out[(size_t)n * out_row + (size_t)h * out_head + j] = from_f32<T>(acc);
  }
}

// One token a sequence over its cached rows (its own among them): q [B, H, R + dr] in the rows' channels, out [B, H, R] =
// the softmax-weighted sum of c.  A workgroup a (sequence, head): the 32-bit path, and any shape.
template <typename T>
__global__ void __launch_bounds__(256)
latent_attn_plain_kernel(const T* __restrict__ q, const T* __restrict__ pages, const int* __restrict__ table, int table_stride,
                         int ring_pages, const int* __restrict__ row_pos, int H, int R, int dr, int window, float scale,
                         T* __restrict__ out) {
  __shared__ float q_s[LC_MAX_R + LC_MAX_ROT];
  __shared__ float p_s[PAGE];
  __shared__ float sh[4];
  const int b = blockIdx.x / H, t = threadIdx.x, lane = t % WAVE, wave = t / WAVE, D = R + dr;
  const int p = row_pos[b];
  const int lo = (window > 0 && p - window + 1 > 0) ? p - window + 1 : 0;
  for (int i = t; i < D; i += 256) q_s[i] = to_f32(q[(size_t)blockIdx.x * D + i]);
  float m = -INFINITY, l = 0.f, acc[LC_MAX_R / 256];
#pragma unroll
  for (int i = 0; i < LC_MAX_R / 256; ++i) acc[i] = 0.f;
  for (int pg = lo / PAGE; pg <= p / PAGE; ++pg) {
    const T* rows = pages + (size_t)table[(size_t)b * table_stride + pg % ring_pages] * PAGE * D;
    const int r0 = max(lo - pg * PAGE, 0), r1 = min(p - pg * PAGE, PAGE - 1);
    __syncthreads();
    for (int r = wave; r < PAGE; r += 4) {
      float s = -INFINITY;
      if (r >= r0 && r <= r1) {
        float dot = 0.f;
        for (int i = lane; i < D; i += WAVE) dot = fmaf(to_f32(rows[(size_t)r * D + i]), q_s[i], dot);
        s = wave_sum(dot) * scale;
      }
      if (lane == 0) p_s[r] = s;
    }
    __syncthreads();
    const float s = t < PAGE ? p_s[t] : -INFINITY;
    const float m_new = fmaxf(m, block_max<256>(s, sh));       // finite: the page holds a visible row
    const float w = t < PAGE ? expf(s - m_new) : 0.f;
    const float alpha = expf(m - m_new);                        // 0 in the first page
    l = l * alpha + block_sum<256>(w, sh);
    m = m_new;
    if (t < PAGE) p_s[t] = w;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < LC_MAX_R / 256; ++i) {
      const int c = t + 256 * i;
      if (c >= R) continue;
      float a = acc[i] * alpha;
      for (int r = r0; r <= r1; ++r) a = fmaf(p_s[r], to_f32(rows[(size_t)r * D + c]), a);
      acc[i] = a;
    }
  }
#pragma unroll
  for (int i = 0; i < LC_MAX_R / 256; ++i) {
    const int c = t + 256 * i;
    if (c < R) out[(size_t)blockIdx.x * R + c] = from_f32<T>(acc[i] / l);
  }
}

}  // namespace tl

using namespace tl;

extern "C" {

// qf: row n's q at qf + n * q_stride; cf: row n's [a (R) | b (dr)] at cf + n * c_stride (floats)
int tl_latent_prepare(const float* qf, int q_stride, const float* cf, int c_stride, int n, int H, int dn, int dr, int R,
                      const float* w, float eps, const int* row_pos, const float* inv_freq, int rotary_dim, int interleaved,
                      float magnitude, void* qn, long long qn_row, long long qn_head, void* qr, long long qr_row,
                      long long qr_head, void* c, void* rows, void* pages, const int* table, int table_stride, int ring_pages,
                      int dt, hipStream_t st) {
  TL_REQUIRE(n >= 0 && H > 0 && dn > 0 && dr >= 0 && dr % 2 == 0 && dr <= LC_MAX_ROT && R > 0,
             "latent_prepare: bad sizes n=%d H=%d dn=%d dr=%d R=%d", n, H, dn, dr, R);
  TL_REQUIRE(q_stride >= H * (dn + dr) && c_stride >= R + dr, "latent_prepare: rows shorter than their parts");
  TL_REQUIRE(rotary_dim >= 0 && rotary_dim % 2 == 0 && rotary_dim <= dr && (rotary_dim == 0 || inv_freq),
             "latent_prepare: %d rotated channels of %d", rotary_dim, dr);
  TL_REQUIRE(qf && cf && w && row_pos && qn && (qr || dr == 0) && (c || rows || pages), "latent_prepare: a buffer is missing");
  TL_REQUIRE(pages == nullptr || (table && table_stride > 0 && ring_pages > 0), "latent_prepare: pages without a page table");
  TL_REQUIRE(dt == DT_F32 || dt == DT_BF16, "latent_prepare: unknown dtype code %d", dt);
  if (n == 0) return 0;
  const Rotation rot{inv_freq, rotary_dim, interleaved, magnitude};
  const dim3 grid(n, 1 + (H + LP_HEADS - 1) / LP_HEADS);
  if (dt == DT_F32) {
    const LatentOut<float> o{(float*)qn, qn_row, qn_head, (float*)qr, qr_row, qr_head, (float*)c, (float*)rows, (float*)pages, table,
                             table_stride, ring_pages};
    latent_prepare_kernel<float><<<grid, 256, 0, st>>>(qf, q_stride, cf, c_stride, H, dn, dr, R, w, eps, row_pos, rot, o);
  } else {
    const LatentOut<bf16> o{(bf16*)qn, qn_row, qn_head, (bf16*)qr, qr_row, qr_head, (bf16*)c, (bf16*)rows, (bf16*)pages, table,
                            table_stride, ring_pages};
    latent_prepare_kernel<bf16><<<grid, 256, 0, st>>>(qf, q_stride, cf, c_stride, H, dn, dr, R, w, eps, row_pos, rot, o);
  }
  TL_LAUNCH_CHECK("latent_prepare");
  return 0;
}

int tl_latent_commit(const void* rows, int dt, const int* row_seq, const int* row_pos, const int* len_after, const int* table,
                     int table_stride, int ring_pages, int n, int D, void* pages, hipStream_t st) {
  TL_REQUIRE(n >= 0 && D > 0 && ring_pages > 0 && table_stride > 0, "latent_commit: bad sizes n=%d D=%d", n, D);
  TL_REQUIRE(rows && row_seq && row_pos && len_after && table && pages, "latent_commit: a buffer is missing");
  TL_REQUIRE(dt == DT_F32 || dt == DT_BF16, "latent_commit: unknown dtype code %d", dt);
  if (n == 0) return 0;
  if (dt == DT_F32)
    latent_commit_kernel<float><<<n, 256, 0, st>>>((const float*)rows, row_seq, row_pos, len_after, table, table_stride, ring_pages,
                                                   D, (float*)pages);
  else
    latent_commit_kernel<bf16><<<n, 256, 0, st>>>((const bf16*)rows, row_seq, row_pos, len_after, table, table_stride, ring_pages, D,
                                                  (bf16*)pages);
  TL_LAUNCH_CHECK("latent_commit");
  return 0;
}

int tl_latent_gather(const void* pages, int dt, const int* table, int table_stride, const int* off, int B, int n_pages, int R,
                     int dr, void* c, void* kr, hipStream_t st) {
  TL_REQUIRE(B > 0 && n_pages >= 0 && R > 0 && dr >= 0 && table_stride > 0, "latent_gather: bad sizes B=%d pages=%d R=%d dr=%d", B,
             n_pages, R, dr);
  TL_REQUIRE(pages && table && off && c && (kr || dr == 0), "latent_gather: a buffer is missing");
  TL_REQUIRE(dt == DT_F32 || dt == DT_BF16, "latent_gather: unknown dtype code %d", dt);
  if (n_pages == 0) return 0;
  const dim3 grid(n_pages, 8);
  if (dt == DT_F32)
    latent_gather_kernel<float><<<grid, 256, 0, st>>>((const float*)pages, table, table_stride, off, B, R, dr, (float*)c, (float*)kr);
  else
    latent_gather_kernel<bf16><<<grid, 256, 0, st>>>((const bf16*)pages, table, table_stride, off, B, R, dr, (bf16*)c, (bf16*)kr);
  TL_LAUNCH_CHECK("latent_gather");
  return 0;
}

// kr: row n's rotated key part at kr + n * kr_stride elements
int tl_latent_heads(const float* kvf, const void* kr, int kr_stride, int n, int H, int dn, int dr, int dv, void* k, void* v, int dt,
                    hipStream_t st) {
  TL_REQUIRE(n >= 0 && H > 0 && dn > 0 && dr >= 0 && dv > 0 && kr_stride >= dr, "latent_heads: bad sizes n=%d H=%d dn=%d dr=%d dv=%d", n,
             H, dn, dr, dv);
  TL_REQUIRE(kvf && (kr || dr == 0) && k && v, "latent_heads: a buffer is missing");
  TL_REQUIRE(dt == DT_F32 || dt == DT_BF16, "latent_heads: unknown dtype code %d", dt);
  if (n == 0) return 0;
  const dim3 grid(n, (H * (dn + dr + dv) + LH_CHUNK - 1) / LH_CHUNK);
  if (dt == DT_F32)
    latent_heads_kernel<float><<<grid, 256, 0, st>>>(kvf, (const float*)kr, kr_stride, H, dn, dr, dv, (float*)k, (float*)v);
  else
    latent_heads_kernel<bf16><<<grid, 256, 0, st>>>(kvf, (const bf16*)kr, kr_stride, H, dn, dr, dv, (bf16*)k, (bf16*)v);
  TL_LAUNCH_CHECK("latent_heads");
  return 0;
}

int tl_latent_heads_pages(const float* kvf, const void* kr, int n_pages, int H, int dn, int dr, int dv, void* out, int dt,
                          hipStream_t st) {
  TL_REQUIRE(n_pages >= 0 && H > 0 && H <= 65535 && dn > 0 && dr >= 0 && dv > 0, "latent_heads_pages: bad sizes pages=%d H=%d dn=%d dr=%d dv=%d",
             n_pages, H, dn, dr, dv);
  TL_REQUIRE(kvf && (kr || dr == 0) && out, "latent_heads_pages: a buffer is missing");
  TL_REQUIRE(dt == DT_F32 || dt == DT_BF16, "latent_heads_pages: unknown dtype code %d", dt);
  if (n_pages == 0) return 0;
  const dim3 grid(n_pages, H);
  if (dt == DT_F32)
    latent_heads_pages_kernel<float><<<grid, 256, 0, st>>>(kvf, (const float*)kr, H, dn, dr, dv, (float*)out);
  else
    latent_heads_pages_kernel<bf16><<<grid, 256, 0, st>>>(kvf, (const bf16*)kr, H, dn, dr, dv, (bf16*)out);
  TL_LAUNCH_CHECK("latent_heads_pages");
  return 0;
}

int tl_head_products(const void* x, const void* w, int n, int H, int N, int K, void* out, long long out_row, long long out_head,
                     int dt, hipStream_t st) {
  TL_REQUIRE(n >= 0 && n <= 65535 && H > 0 && H <= 65535 && N > 0 && K > 0 && out_head >= N, "head_products: bad sizes n=%d H=%d N=%d K=%d", n,
             H, N, K);
  TL_REQUIRE(x && w && out, "head_products: a buffer is missing");
  TL_REQUIRE(dt == DT_F32 || dt == DT_BF16, "head_products: unknown dtype code %d", dt);
  if (n == 0) return 0;
  const dim3 grid((N + 31) / 32, H, n);
  if (dt == DT_F32)
    head_products_kernel<float><<<grid, 256, 0, st>>>((const float*)x, (const float*)w, H, N, K, (float*)out, out_row, out_head);
  else
    head_products_kernel<bf16><<<grid, 256, 0, st>>>((const bf16*)x, (const bf16*)w, H, N, K, (bf16*)out, out_row, out_head);
  TL_LAUNCH_CHECK("head_products");
  return 0;
}

int tl_latent_attn_plain(const void* q, const void* pages, int dt, const int* table, int table_stride, int ring_pages,
                         const int* row_pos, int B, int H, int R, int dr, int window, float scale, void* out, hipStream_t st) {
  TL_REQUIRE(B >= 0 && H > 0 && R > 0 && R <= LC_MAX_R && dr >= 0 && dr <= LC_MAX_ROT && window >= 0,
             "latent attention: bad sizes B=%d H=%d R=%d dr=%d window=%d", B, H, R, dr, window);
  TL_REQUIRE(q && pages && table && row_pos && out && table_stride > 0 && ring_pages > 0, "latent attention: a buffer is missing");
  TL_REQUIRE(dt == DT_F32 || dt == DT_BF16, "latent attention: unknown dtype code %d", dt);
  TL_REQUIRE((long long)B * H < 2147483647LL, "latent attention: too many (row, head) pairs");
  if (B == 0) return 0;
  if (dt == DT_F32)
    latent_attn_plain_kernel<float><<<B * H, 256, 0, st>>>((const float*)q, (const float*)pages, table, table_stride, ring_pages,
                                                           row_pos, H, R, dr, window, scale, (float*)out);
  else
    latent_attn_plain_kernel<bf16><<<B * H, 256, 0, st>>>((const bf16*)q, (const bf16*)pages, table, table_stride, ring_pages, row_pos,
                                                          H, R, dr, window, scale, (bf16*)out);
  TL_LAUNCH_CHECK("latent_attn_plain");
  return 0;
}

}  // extern "C"
