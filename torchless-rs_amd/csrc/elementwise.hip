// Row-wise kernels: embedding gather, RMSNorm, rotation + split of the fused
// q|k|v projection, commit of keys and values to cache pages, SiLU-gate,
// row gather.  Reductions, angles and the norm are computed in float.
#include "common.hpp"
#include <stdarg.h>

namespace tl {

static thread_local char g_err[512] = "";
void set_error(const char* fmt, ...) {
  va_list ap;
  va_start(ap, fmt);
  vsnprintf(g_err, sizeof(g_err), fmt, ap);
  va_end(ap);
}

// ---- embedding: out[n, :] = table[ids[n], :] * scale ---------------------------
// src/model/modules/embedding.rs:15-21 of the reference (which has no scaling: scale 1).
template <typename T>
__global__ void embed_kernel(const T* __restrict__ table, const int* __restrict__ ids, int H, float scale,
                             float* __restrict__ out) {
  const int n = blockIdx.x;
  const T* row = table + (size_t)ids[n] * H;
  float* o = out + (size_t)n * H;
  for (int i = threadIdx.x; i < H; i += blockDim.x) o[i] = to_f32(row[i]) * scale;
}

// The same with a second table read by pairs of tokens, and a norm of the sum: row (previous * mul_prev + current * mul_cur)
// mod buckets of `pairs`, row `buckets` for a sequence's first token.  The previous token of a sequence's first row of the
// step lies in `last`; the workgroup of that row alone reads and then replaces it.  One workgroup a row, which stays in
// registers (IT > 0: H % 4 == 0, H <= 1024 * IT) or goes through `out` (every thread reads back what it wrote).
struct PairTerms {
  const int* row_pos;
  const int* row_seq;
  const int* cu_seqlens;
  const int* slots;
  int* last;
  long long buckets, mul_prev, mul_cur;
};
__device__ __forceinline__ f32x4 row4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ f32x4 row4(const bf16* p) {
  const bf16x4 v = *reinterpret_cast<const bf16x4*>(p);
  return f32x4{(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
}
template <typename T, int IT>
__global__ void __launch_bounds__(256)
embed_pairs_kernel(const T* __restrict__ table, const int* __restrict__ ids, int H, float scale, const T* __restrict__ pairs, PairTerms k,
                   const float* __restrict__ w, float eps, float* __restrict__ out) {
  __shared__ float sh[4];
  __shared__ int s_prev;
  const int n = blockIdx.x;
  const T* row = table + (size_t)ids[n] * H;
  constexpr int R = IT > 0 ? IT : 1;
  f32x4 v[R], wv[R];                                   // (asked for before the previous token is known)
  if constexpr (IT > 0) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int i = (threadIdx.x + 256 * r) * 4;
      if (i < H) {
        v[r] = row4(row + i);
        if (w) wv[r] = *reinterpret_cast<const f32x4*>(w + i);
      }
    }
  }
  const T* second = nullptr;
  if (pairs) {
    if (threadIdx.x == 0) {
      const int b = k.row_seq[n], before = n > 0 ? ids[n - 1] : -1, pos = k.row_pos[n];
      const int row0 = k.cu_seqlens[b], end = k.cu_seqlens[b + 1], slot = k.slots[b];
      int prev = before;
      if (n == row0) {
        prev = k.last[slot];
        k.last[slot] = ids[end - 1];
      }
      s_prev = pos == 0 ? -1 : prev;
    }
    __syncthreads();
    const int prev = s_prev;
    // (two products of 31 bits each fit 63)
    const long long at = prev < 0 ? k.buckets : (prev * k.mul_prev + ids[n] * k.mul_cur) % k.buckets;
    second = pairs + (size_t)at * H;
  }
  float* o = out + (size_t)n * H;
  float ss = 0.f;
  if constexpr (IT > 0) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int i = (threadIdx.x + 256 * r) * 4;
      if (i >= H) continue;
      v[r] *= scale;
      if (second) v[r] += row4(second + i);
      ss += v[r][0] * v[r][0] + v[r][1] * v[r][1] + v[r][2] * v[r][2] + v[r][3] * v[r][3];
    }
    if (w) ss = block_sum<256>(ss, sh);
    const float root = sqrtf(ss / (float)H + eps);
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int i = (threadIdx.x + 256 * r) * 4;
      if (i >= H) continue;
      if (w)
#pragma unroll
        for (int e = 0; e < 4; ++e) v[r][e] = (v[r][e] / root) * wv[r][e];
      *reinterpret_cast<f32x4*>(o + i) = v[r];
    }
    return;
  }
  for (int i = threadIdx.x; i < H; i += 256) {
    float a = to_f32(row[i]) * scale;
    if (second) a += to_f32(second[i]);
    o[i] = a;
    ss += a * a;
  }
  if (w == nullptr) return;
  ss = block_sum<256>(ss, sh);
  const float rms = sqrtf(ss / (float)H + eps);
  for (int i = threadIdx.x; i < H; i += 256) o[i] = (o[i] / rms) * w[i];
}

// ---- RMSNorm: y = x / sqrt(mean(x^2) + eps) * w ------------------------------
// src/kernels/mod.rs:558-568 of the reference: eps inside the root, divide,
// then multiply by the weight.
template <typename TO>
__global__ void __launch_bounds__(256) rmsnorm_kernel(const float* __restrict__ x,
                                                      const float* __restrict__ w, float eps,
                                                      TO* __restrict__ out, int H) {
  __shared__ float sh[4];
  const int n = blockIdx.x;
  const float* xr = x + (size_t)n * H;
  float ss = 0.f;
  for (int i = threadIdx.x; i < H; i += 256) {
    float v = xr[i];
    ss += v * v;
  }
  ss = block_sum<256>(ss, sh);
  const float rms = sqrtf(ss / (float)H + eps);
  TO* o = out + (size_t)n * H;
  for (int i = threadIdx.x; i < H; i += 256) o[i] = from_f32<TO>((xr[i] / rms) * w[i]);
}

// The same with the row held in registers: one read of x.  H % 4 == 0, H <= 1024 * IT.
template <typename TO, int IT>
__global__ void __launch_bounds__(256) rmsnorm_reg_kernel(const float* __restrict__ x,
                                                          const float* __restrict__ w, float eps,
                                                          TO* __restrict__ out, int H) {
  __shared__ float sh[4];
  const int n = blockIdx.x;
  const float4* xr = reinterpret_cast<const float4*>(x + (size_t)n * H);
  const float4* wr = reinterpret_cast<const float4*>(w);
  const int nv = H / 4;
  float4 v[IT], g[IT];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < IT; ++i) {
    const int c = threadIdx.x + 256 * i;
    if (c < nv) {
      v[i] = xr[c];
      g[i] = wr[c];
      ss += v[i].x * v[i].x + v[i].y * v[i].y + v[i].z * v[i].z + v[i].w * v[i].w;
    }
  }
  ss = block_sum<256>(ss, sh);
  const float rms = sqrtf(ss / (float)H + eps);
  TO* o = out + (size_t)n * H;
#pragma unroll
  for (int i = 0; i < IT; ++i) {
    const int c = threadIdx.x + 256 * i;
    if (c < nv) {
      o[4 * c + 0] = from_f32<TO>((v[i].x / rms) * g[i].x);
      o[4 * c + 1] = from_f32<TO>((v[i].y / rms) * g[i].y);
      o[4 * c + 2] = from_f32<TO>((v[i].z / rms) * g[i].z);
      o[4 * c + 3] = from_f32<TO>((v[i].w / rms) * g[i].w);
    }
  }
}

// x += sum of the partial products P[s][n][H] (in the order of s), then the norm of the new x.
template <typename TO, int IT>
__global__ void __launch_bounds__(256)
add_rmsnorm_reg_kernel(float* __restrict__ x, const float* __restrict__ parts, int n_parts, size_t part_stride,
                       const float* __restrict__ w, float eps, TO* __restrict__ out, int H) {
  __shared__ float sh[4];
  const int n = blockIdx.x;
  float4* xr = reinterpret_cast<float4*>(x + (size_t)n * H);
  const float4* wr = reinterpret_cast<const float4*>(w);
  const int nv = H / 4;
  float4 v[IT], g[IT];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < IT; ++i) {
    const int c = threadIdx.x + 256 * i;
    if (c < nv) {
      float4 a = xr[c];
#pragma unroll 4
      for (int s = 0; s < n_parts; ++s) {
        const float4 p = reinterpret_cast<const float4*>(parts + s * part_stride + (size_t)n * H)[c];
        a.x += p.x; a.y += p.y; a.z += p.z; a.w += p.w;
      }
      xr[c] = a;
      v[i] = a;
      g[i] = wr[c];
      ss += a.x * a.x + a.y * a.y + a.z * a.z + a.w * a.w;
    }
  }
  ss = block_sum<256>(ss, sh);
  const float rms = sqrtf(ss / (float)H + eps);
  TO* o = out + (size_t)n * H;
#pragma unroll
  for (int i = 0; i < IT; ++i) {
    const int c = threadIdx.x + 256 * i;
    if (c < nv) {
      o[4 * c + 0] = from_f32<TO>((v[i].x / rms) * g[i].x);
      o[4 * c + 1] = from_f32<TO>((v[i].y / rms) * g[i].y);
      o[4 * c + 2] = from_f32<TO>((v[i].z / rms) * g[i].z);
      o[4 * c + 3] = from_f32<TO>((v[i].w / rms) * g[i].w);
    }
  }
}

__global__ void add_partials_kernel(float* __restrict__ x, const float* __restrict__ parts, int n_parts,
                                    size_t part_stride, size_t total) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= total) return;
  float a = x[i];
  for (int s = 0; s < n_parts; ++s) a += parts[s * part_stride + i];
  x[i] = a;
}

// ---- rotation and split ------------------------------------------------------
// qkv[n, :] = [q (nq*d) | k (nkv*d) | v (nkv*d)] in float.  q and k are rotated
// in pairs by the angle pos * inv_freq[i] (which channels make pair i, and how many
// of a head's channels are rotated: `Rotation`, `pair_channels`); v is copied.
// The reference rotates all channels in pairs (i, i + d/2):
// src/kernels/mod.rs:582-608, src/model/modules/attention.rs:68-78.
constexpr int ROPE_MAX_HALF = 128;      // head sizes up to 256

template <typename TO>
__device__ __forceinline__ void rope_split_row(int n, float* cs, float* sn, const float* __restrict__ qkv,
                                               const int* __restrict__ row_pos, Rotation rot, int nq, int nkv, int d,
                                               TO* __restrict__ q, TO* __restrict__ k, TO* __restrict__ v,
                                               TO* __restrict__ vt, int vt_cols, const int* __restrict__ row_seq,
                                               const int* __restrict__ tile_off, const int* __restrict__ n_cached) {
  const int half = d / 2, rot_pairs = rot.rotary_dim / 2;
  const float pos = (float)row_pos[n];
  for (int i = threadIdx.x; i < rot_pairs; i += blockDim.x) {     // the row's angles, once
    const float ang = rot.inv_freq[i] * pos;
    sincosf(ang, &sn[i], &cs[i]);          // one routine for both, the same in every kernel that rotates
  }
  __syncthreads();
  const float* src = qkv + (size_t)n * (nq + 2 * nkv) * d;
  const int n_rot = (nq + nkv) * half;
  for (int t = threadIdx.x; t < n_rot; t += blockDim.x) {
    const int h = t / half, i = t % half;
    int ia, ib;
    pair_channels(i, rot.rotary_dim, rot.interleaved, ia, ib);
    const float a = src[h * d + ia], b = src[h * d + ib];
    float ra = a, rb = b;
    if (i < rot_pairs) rotate_pair(a, b, cs[i], sn[i], ra, rb);
    TO* dst = (h < nq) ? q + ((size_t)n * nq + h) * d : k + ((size_t)n * nkv + (h - nq)) * d;
    dst[ia] = from_f32<TO>(ra);
    dst[ib] = from_f32<TO>(rb);
  }
  const float* vs = src + (size_t)(nq + nkv) * d;
  if (v != nullptr) {
    TO* vd = v + (size_t)n * nkv * d;
    for (int t = threadIdx.x; t < nkv * d; t += blockDim.x) vd[t] = from_f32<TO>(vs[t]);
  }
  if (vt != nullptr) {      // the same values transposed: [kv head][d][column of this row]
    const int b = row_seq[n];
    const int col = tile_off[b] + row_pos[n] - (n_cached[b] / PAGE) * PAGE;
    for (int t = threadIdx.x; t < nkv * d; t += blockDim.x) vt[(size_t)t * vt_cols + col] = from_f32<TO>(vs[t]);
  }
}

template <typename TO>
__global__ void rope_split_kernel(const float* __restrict__ qkv, const int* __restrict__ row_pos,
                                  Rotation rot, int nq, int nkv, int d,
                                  TO* __restrict__ q, TO* __restrict__ k, TO* __restrict__ v,
                                  TO* __restrict__ vt, int vt_cols, const int* __restrict__ row_seq,
                                  const int* __restrict__ tile_off, const int* __restrict__ n_cached) {
  __shared__ float cs[ROPE_MAX_HALF], sn[ROPE_MAX_HALF];
  rope_split_row<TO>(blockIdx.x, cs, sn, qkv, row_pos, rot, nq, nkv, d, q, k, v, vt, vt_cols, row_seq, tile_off,
                     n_cached);
}

// ---- commit keys and values of this step to the pages -----------------------
// Position p of sequence b goes to page table[b][(p / PAGE) % ring_pages], row
// p % PAGE.  Rows that would be overwritten within this same step (older than
// the last ring_pages * PAGE positions) are skipped.  A page holds, per KV
// head, keys as [PAGE][d] and values transposed as [d][PAGE], so that both
// are read along their contraction index by the matrix cores.
template <typename T>
__global__ void kv_commit_kernel(const T* __restrict__ k, const T* __restrict__ v,
                                 const int* __restrict__ row_seq, const int* __restrict__ row_pos,
                                 const int* __restrict__ len_after, const int* __restrict__ table,
                                 int table_stride, int ring_pages, int nkv, int d,
                                 T* __restrict__ pages) {
  const int n = blockIdx.x;
  const int b = row_seq[n], p = row_pos[n];
  if (p < len_after[b] - ring_pages * PAGE) return;
  const int page = table[(size_t)b * table_stride + (p / PAGE) % ring_pages];
  const int r = p % PAGE;
  const size_t page_elems = (size_t)2 * nkv * PAGE * d;
  T* kd = pages + (size_t)page * page_elems;
  T* vd = kd + (size_t)nkv * PAGE * d;
  const T* ks = k + (size_t)n * nkv * d;
  const T* vs = v + (size_t)n * nkv * d;
  for (int t = threadIdx.x; t < nkv * d; t += blockDim.x) {
    const int h = t / d, i = t % d;
    kd[((size_t)h * PAGE + r) * d + i] = ks[t];
    vd[((size_t)h * d + i) * PAGE + r] = vs[t];
  }
}

// ---- values by tiles of 64 positions ------------------------------------------
// Buffers laid out by aligned columns hold sequence b from column tile_off[b] on, position
// 64 * (n_cached[b] / 64) first, so that a tile of 64 columns is one cache page.  Which
// sequence and which positions a tile of columns holds:
struct ColumnTile {
  int b, p0, lo, hi;        // sequence, position of column 0, positions [lo, hi) of this step in it
};
__device__ __forceinline__ ColumnTile column_tile(int col0, int B, const int* tile_off, const int* n_cached,
                                                  const int* len_after) {
  int b = 0;
  while (b + 1 < B && tile_off[b + 1] <= col0) ++b;
  const int cached = n_cached[b], after = len_after[b];
  ColumnTile t;
  t.b = b;
  t.p0 = (cached / PAGE) * PAGE + (col0 - tile_off[b]);
  t.lo = max(t.p0, cached);
  t.hi = min(t.p0 + PAGE, after);            // lo >= hi: padding, nothing of this step
  return t;
}

// vt[kv head][dv][column] = v of the row at that column, from the fused projection (float):
// the transposed values of a step, written in whole lines (a row-by-row kernel writes them
// two bytes at a time, a line apart).  grid: (columns / 64, kv heads, d / 64 rounded up).
template <typename TO, typename TS = float>       // TS: the type of the rows the values are read from
__device__ __forceinline__ void v_tile(int col_block, int kvh, int d_block, TO (*tile)[PAGE + 2],
                                       const TS* __restrict__ qkv, int width, int v_off, int d,
                                       TO* __restrict__ vt, int vt_cols, int B, const int* __restrict__ cu_seqlens,
                                       const int* __restrict__ tile_off, const int* __restrict__ n_cached,
                                       const int* __restrict__ len_after) {
  const int col0 = col_block * PAGE;
  const ColumnTile t = column_tile(col0, B, tile_off, n_cached, len_after);
  if (t.lo >= t.hi) return;
  const int row0 = cu_seqlens[t.b] - n_cached[t.b];       // row of position p is row0 + p
  const int c0 = d_block * 64, dc = min(64, d - c0);       // this block's 64 of the d values
  // all loads first (16 a thread), then the stores: one trip to memory
  float tmp[16];
#pragma unroll
  for (int u = 0; u < 16; ++u) {
    const int idx = threadIdx.x + 256 * u;
    const int r = idx / dc, i = idx % dc, p = t.p0 + r;
    tmp[u] = (idx < PAGE * dc && p >= t.lo && p < t.hi)
                 ? to_f32(qkv[(size_t)(row0 + p) * width + v_off + kvh * d + c0 + i]) : 0.f;
  }
#pragma unroll
  for (int u = 0; u < 16; ++u) {
    const int idx = threadIdx.x + 256 * u;
    if (idx < PAGE * dc) tile[idx % dc][idx / dc] = from_f32<TO>(tmp[u]);
  }
  __syncthreads();
#pragma unroll
  for (int u = 0; u < 16; ++u) {
    const int idx = threadIdx.x + 256 * u;
    const int i = idx / PAGE, r = idx % PAGE, p = t.p0 + r;
    if (i < dc && p >= t.lo && p < t.hi) vt[((size_t)kvh * d + c0 + i) * vt_cols + col0 + r] = tile[i][r];
  }
}

template <typename TO, typename TS = float>
__global__ void __launch_bounds__(256)
v_tiles_kernel(const TS* __restrict__ qkv, int width, int v_off, int d, TO* __restrict__ vt,
               int vt_cols, int B, const int* __restrict__ cu_seqlens, const int* __restrict__ tile_off,
               const int* __restrict__ n_cached, const int* __restrict__ len_after) {
  __shared__ TO tile[64][PAGE + 2];
  v_tile<TO, TS>(blockIdx.x, blockIdx.y, blockIdx.z, tile, qkv, width, v_off, d, vt, vt_cols, B, cu_seqlens, tile_off,
             n_cached, len_after);
}

// Both of the above in one launch, for a step with several rows a sequence: the first n workgroups
// rotate a row each (q and k; the values are the tiles' business), the others transpose a tile of
// values each.  The two read the same buffer and write different ones.
template <typename TO>
__global__ void __launch_bounds__(256)
rope_v_tiles_kernel(const float* __restrict__ qkv, const int* __restrict__ row_pos, Rotation rot, int n, int nq,
                    int nkv, int d, TO* __restrict__ q, TO* __restrict__ k, TO* __restrict__ vt, int vt_cols, int B,
                    const int* __restrict__ cu_seqlens, const int* __restrict__ tile_off,
                    const int* __restrict__ n_cached, const int* __restrict__ len_after) {
  __shared__ __attribute__((aligned(16))) unsigned char sh[sizeof(TO) * 64 * (PAGE + 2) > 2 * sizeof(float) * ROPE_MAX_HALF
                                                            ? sizeof(TO) * 64 * (PAGE + 2)
                                                            : 2 * sizeof(float) * ROPE_MAX_HALF];
  if ((int)blockIdx.x < n) {
    float* cs = reinterpret_cast<float*>(sh);
    rope_split_row<TO>(blockIdx.x, cs, cs + ROPE_MAX_HALF, qkv, row_pos, rot, nq, nkv, d, q, k, (TO*)nullptr,
                       (TO*)nullptr, 0, nullptr, nullptr, nullptr);
    return;
  }
  const int item = blockIdx.x - n, d_blocks = (d + 63) / 64;
  const int d_block = item % d_blocks, kvh = (item / d_blocks) % nkv, col_block = item / (d_blocks * nkv);
  v_tile<TO>(col_block, kvh, d_block, reinterpret_cast<TO(*)[PAGE + 2]>(sh), qkv, (nq + 2 * nkv) * d, (nq + nkv) * d, d,
             vt, vt_cols, B, cu_seqlens, tile_off, n_cached, len_after);
}

// Commit of a step whose values lie transposed by tiles: the first blocks put the keys of 8 rows
// each into their pages, the others copy a tile of values [d][64] of one KV head in whole lines.
// Positions that the same step overwrites in a ring are skipped, as in kv_commit.
template <typename T>
__global__ void __launch_bounds__(256)
kv_commit_tiles_kernel(const T* __restrict__ k, const T* __restrict__ vt, int vt_cols, int n,
                       const int* __restrict__ row_seq, const int* __restrict__ row_pos, int B,
                       const int* __restrict__ tile_off, const int* __restrict__ n_cached,
                       const int* __restrict__ len_after, const int* __restrict__ table, int table_stride,
                       int ring_pages, int nkv, int d, T* __restrict__ pages) {
  const size_t page_elems = (size_t)2 * nkv * PAGE * d;
  const int k_blocks = (n + 7) / 8;
  if ((int)blockIdx.x < k_blocks) {
    // 8 rows a block, 32 threads a row, 16 bytes at a time where the head size allows
    constexpr int VEC = 16 / sizeof(T);
    const int r_n = blockIdx.x * 8 + threadIdx.x / 32, lane = threadIdx.x % 32;
    if (r_n >= n) return;
    const int b = row_seq[r_n], p = row_pos[r_n];
    if (p < len_after[b] - ring_pages * PAGE) return;
    const int page = table[(size_t)b * table_stride + (p / PAGE) % ring_pages];
    T* kd = pages + (size_t)page * page_elems;
    const T* ks = k + (size_t)r_n * nkv * d;
    if (d % VEC == 0 && ((uintptr_t)k % 16 == 0) && ((uintptr_t)pages % 16 == 0)) {
      for (int c = lane; c < nkv * d / VEC; c += 32) {
        const int e = c * VEC, h = e / d, i = e % d;
        *reinterpret_cast<f32x4*>(&kd[((size_t)h * PAGE + p % PAGE) * d + i]) =
            *reinterpret_cast<const f32x4*>(&ks[e]);
      }
    } else {
      for (int t = lane; t < nkv * d; t += 32) {
        const int h = t / d, i = t % d;
        kd[((size_t)h * PAGE + p % PAGE) * d + i] = ks[t];
      }
    }
    return;
  }
  const int v_block = blockIdx.x - k_blocks;
  const int col0 = (v_block / nkv) * PAGE, kvh = v_block % nkv;
  const ColumnTile t = column_tile(col0, B, tile_off, n_cached, len_after);
  const int lo = max(t.lo, len_after[t.b] - ring_pages * PAGE);
  if (lo >= t.hi) return;
  const int page = table[(size_t)t.b * table_stride + (t.p0 / PAGE) % ring_pages];
  T* vd = pages + (size_t)page * page_elems + (size_t)nkv * PAGE * d + (size_t)kvh * d * PAGE;
  const T* vs = vt + (size_t)kvh * d * vt_cols + col0;
  for (int base = 0; base < d * PAGE; base += 256 * 16) {      // 16 loads a thread, then their stores
    T tmp[16];
#pragma unroll
    for (int u = 0; u < 16; ++u) {
      const int idx = base + threadIdx.x + 256 * u;
      const int i = idx / PAGE, r = idx % PAGE, p = t.p0 + r;
      if (i < d && p >= lo && p < t.hi) tmp[u] = vs[(size_t)i * vt_cols + r];
    }
#pragma unroll
    for (int u = 0; u < 16; ++u) {
      const int idx = base + threadIdx.x + 256 * u;
      const int i = idx / PAGE, r = idx % PAGE, p = t.p0 + r;
      if (i < d && p >= lo && p < t.hi) vd[(size_t)i * PAGE + r] = tmp[u];
    }
  }
}

// ---- single-token steps: rotate, and put k and v straight into the pages ------
// Row n is the one new token of sequence n (position row_pos[n]).
// qkv may come as n_parts partial products (part_stride elements apart) that are added up here.
template <typename T>
__global__ void rope_commit_kernel(const float* __restrict__ qkv, int n_parts, size_t part_stride,
                                   const int* __restrict__ row_pos,
                                   Rotation rot, const int* __restrict__ table,
                                   int table_stride, int ring_pages, int nq, int nkv, int d,
                                   T* __restrict__ q, T* __restrict__ pages) {
  // blockIdx.y of gridDim.y takes its share of the (q and k) heads and of the values
  __shared__ float cs[ROPE_MAX_HALF], sn[ROPE_MAX_HALF];
  const int n = blockIdx.x;
  const int half = d / 2, rot_pairs = rot.rotary_dim / 2;
  const int p = row_pos[n];
  const float pos = (float)p;
  const float* src = qkv + (size_t)n * (nq + 2 * nkv) * d;
  const int page = table[(size_t)n * table_stride + (p / PAGE) % ring_pages];
  const int r = p % PAGE;
  T* kd = pages + (size_t)page * 2 * nkv * PAGE * d;
  T* vd = kd + (size_t)nkv * PAGE * d;
  for (int i = threadIdx.x; i < rot_pairs; i += blockDim.x) {
    const float ang = rot.inv_freq[i] * pos;
    sincosf(ang, &sn[i], &cs[i]);          // one routine for both, the same in every kernel that rotates
  }
  __syncthreads();
  const int heads = nq + nkv;
  const int h_lo = (int)((long long)heads * blockIdx.y / gridDim.y), h_hi = (int)((long long)heads * (blockIdx.y + 1) / gridDim.y);
  for (int t = h_lo * half + threadIdx.x; t < h_hi * half; t += blockDim.x) {
    const int h = t / half, i = t % half;
    int ia, ib;
    pair_channels(i, rot.rotary_dim, rot.interleaved, ia, ib);
    float a = src[h * d + ia], b = src[h * d + ib];
#pragma unroll 4
    for (int sp = 1; sp < n_parts; ++sp) {
      a += src[sp * part_stride + h * d + ia];
      b += src[sp * part_stride + h * d + ib];
    }
    float ra = a, rb = b;
    if (i < rot_pairs) rotate_pair(a, b, cs[i], sn[i], ra, rb);
    T* dst = (h < nq) ? q + ((size_t)n * nq + h) * d : kd + ((size_t)(h - nq) * PAGE + r) * d;
    dst[ia] = from_f32<T>(ra);
    dst[ib] = from_f32<T>(rb);
  }
  const float* vs = src + (size_t)(nq + nkv) * d;
  const int v_lo = (int)((long long)nkv * d * blockIdx.y / gridDim.y), v_hi = (int)((long long)nkv * d * (blockIdx.y + 1) / gridDim.y);
  for (int t = v_lo + threadIdx.x; t < v_hi; t += blockDim.x) {
    float a = vs[t];
#pragma unroll 4
    for (int sp = 1; sp < n_parts; ++sp) a += vs[sp * part_stride + t];
    vd[(size_t)t * PAGE + r] = from_f32<T>(a);
  }
}

// ---- the function of a gated feed-forward's gate ---------------------------------
// 0: silu(g) = g / (1 + exp(-g)); 1: the tanh form of gelu,
// 0.5 g (1 + tanh(sqrt(2/pi) (g + 0.044715 g^3)))
constexpr int ACT_SILU = 0;
constexpr int ACT_GELU_TANH = 1;
constexpr int ACT_SWISH_CLAMPED = 2;   // g' = min(g, limit), u' = clamp(u, -limit, limit): g' logistic(alpha g') (u' + shift)
constexpr int ACT_RELU = 3;            // max(g, 0)
__device__ __forceinline__ float gate_act(float g, int act) {
  if (act == ACT_RELU) return fmaxf(g, 0.f);
  if (act == ACT_GELU_TANH) return 0.5f * g * (1.0f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)));
  return g / (1.0f + expf(-g));
}
// act(gate) * up with the constants of the functions that have some
struct ActConstants {
  float alpha, limit, shift;
};
__device__ __forceinline__ float gate_times_up(float g, float u, int act, ActConstants k) {
  if (act == ACT_SWISH_CLAMPED) {
    g = fminf(g, k.limit);
    u = fminf(fmaxf(u, -k.limit), k.limit);
    return (g / (1.0f + expf(-k.alpha * g))) * (u + k.shift);
  }
  return gate_act(g, act) * u;
}

// ---- h = silu(gate) * up, silu(g) = g / (1 + exp(-g)) ------------------------
// src/kernels/mod.rs:546-548, src/model/modules/mlp.rs:33-39.
template <typename TO>
__global__ void silu_mul_kernel(const float* __restrict__ gu, int I, TO* __restrict__ out) {
  const int n = blockIdx.x;
  const float* row = gu + (size_t)n * 2 * I;
  for (int i = threadIdx.x; i < I; i += blockDim.x) {
    const float g = row[i], u = row[I + i];
    out[(size_t)n * I + i] = from_f32<TO>((g / (1.0f + expf(-g))) * u);
  }
}

// gu[n, 2I] in bfloat16 with columns in groups of 64 (32 of gate, then the 32 of up
// that belong to them); out[n, I] = silu(gate) * up.  A thread takes 8 pairs.
__global__ void silu_mul_pairs_kernel(const bf16* __restrict__ gu, long long chunks, int I,
                                      bf16* __restrict__ out, int act = ACT_SILU, ActConstants k = ActConstants{1.f, 0.f, 0.f}) {
  const long long c = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= chunks) return;
  const int per_row = I / 8;
  const long long n = c / per_row;
  const int i = (int)(c % per_row), group = i / 4, part = i % 4;
  const bf16* src = gu + n * 2 * I + group * 64 + part * 8;
  const bf16x8 g = *reinterpret_cast<const bf16x8*>(src);
  const bf16x8 u = *reinterpret_cast<const bf16x8*>(src + 32);
  bf16x8 o;
#pragma unroll
  for (int t = 0; t < 8; ++t) {
    const float gv = (float)g[t];
    o[t] = (bf16)gate_times_up(gv, (float)u[t], act, k);
  }
  *reinterpret_cast<bf16x8*>(out + n * I + group * 32 + part * 8) = o;
}

// ---- layer norm with a weight and an optional bias: y = (x - mean) / sqrt(var + eps) * w + beta ----
// var is the mean of the squared deviations from the mean (two passes over the row, both in
// float).  The row may get a bias first (z + b, the bias of the product that made z).
// `x` null: y is written to `out`.  `x` given: the norm is ADDED to the stream, x += y, and
// `out` (may be null) receives the new x in the compute type, for the product that reads
// the stream next.
template <typename TO>
__global__ void __launch_bounds__(256)
layernorm_kernel(const float* __restrict__ z, const float* __restrict__ bias, const float* __restrict__ w,
                 const float* __restrict__ beta, float eps, float* __restrict__ x, TO* __restrict__ out, int H) {
  __shared__ float sh[4];
  const int n = blockIdx.x;
  const float* zr = z + (size_t)n * H;
  float s = 0.f;
  for (int i = threadIdx.x; i < H; i += 256) s += zr[i] + (bias ? bias[i] : 0.f);
  const float mean = block_sum<256>(s, sh) / (float)H;
  float ss = 0.f;
  for (int i = threadIdx.x; i < H; i += 256) {
    const float d = zr[i] + (bias ? bias[i] : 0.f) - mean;
    ss += d * d;
  }
  const float sd = sqrtf(block_sum<256>(ss, sh) / (float)H + eps);
  for (int i = threadIdx.x; i < H; i += 256) {
    const float y = ((zr[i] + (bias ? bias[i] : 0.f) - mean) / sd) * w[i] + (beta ? beta[i] : 0.f);
    if (x) {
      const float xn = x[(size_t)n * H + i] + y;
      x[(size_t)n * H + i] = xn;
      if (out) out[(size_t)n * H + i] = from_f32<TO>(xn);
    } else {
      out[(size_t)n * H + i] = from_f32<TO>(y);
    }
  }
}

// The same with the row held in registers: one read of z.  H % 4 == 0, H <= 1024 * IT.
template <typename TO, int IT>
__global__ void __launch_bounds__(256)
layernorm_reg_kernel(const float* __restrict__ z, const float* __restrict__ bias, const float* __restrict__ w,
                     const float* __restrict__ beta, float eps, float* __restrict__ x, TO* __restrict__ out, int H) {
  __shared__ float sh[4];
  const int n = blockIdx.x;
  const float4* zr = reinterpret_cast<const float4*>(z + (size_t)n * H);
  const float4* br = reinterpret_cast<const float4*>(bias);
  const float4* wr = reinterpret_cast<const float4*>(w);
  const int nv = H / 4;
  float4 v[IT];
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < IT; ++i) {
    const int c = threadIdx.x + 256 * i;
    if (c < nv) {
      v[i] = zr[c];
      if (bias) {
        const float4 b = br[c];
        v[i].x += b.x; v[i].y += b.y; v[i].z += b.z; v[i].w += b.w;
      }
      s += (v[i].x + v[i].y) + (v[i].z + v[i].w);
    }
  }
  const float mean = block_sum<256>(s, sh) / (float)H;
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < IT; ++i) {
    const int c = threadIdx.x + 256 * i;
    if (c < nv) {
      v[i].x -= mean; v[i].y -= mean; v[i].z -= mean; v[i].w -= mean;
      ss += v[i].x * v[i].x + v[i].y * v[i].y + v[i].z * v[i].z + v[i].w * v[i].w;
    }
  }
  const float sd = sqrtf(block_sum<256>(ss, sh) / (float)H + eps);
#pragma unroll
  for (int i = 0; i < IT; ++i) {
    const int c = threadIdx.x + 256 * i;
    if (c < nv) {
      const float4 g = wr[c];
      float4 y;
      y.x = (v[i].x / sd) * g.x; y.y = (v[i].y / sd) * g.y; y.z = (v[i].z / sd) * g.z; y.w = (v[i].w / sd) * g.w;
      if (beta) {
        const float4 e = reinterpret_cast<const float4*>(beta)[c];
        y.x += e.x; y.y += e.y; y.z += e.z; y.w += e.w;
      }
      if (x) {
        float4* xr = reinterpret_cast<float4*>(x + (size_t)n * H);
        float4 a = xr[c];
        a.x += y.x; a.y += y.y; a.z += y.z; a.w += y.w;
        xr[c] = a;
        y = a;
        if (!out) continue;
      }
      TO* o = out + (size_t)n * H + 4 * c;
      o[0] = from_f32<TO>(y.x); o[1] = from_f32<TO>(y.y); o[2] = from_f32<TO>(y.z); o[3] = from_f32<TO>(y.w);
    }
  }
}

// out = x in bfloat16, for a product that reads the stream itself
__global__ void cast_rows_kernel(const float* __restrict__ x, size_t total, bf16* __restrict__ out) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < total) out[i] = (bf16)x[i];
}

// h = act(gate) * up from gu[n, 2I] = [gate | up]
template <typename TO>
__global__ void act_mul_kernel(const float* __restrict__ gu, int I, int act, ActConstants k, TO* __restrict__ out) {
  const int n = blockIdx.x;
  const float* row = gu + (size_t)n * 2 * I;
  for (int i = threadIdx.x; i < I; i += blockDim.x)
    out[(size_t)n * I + i] = from_f32<TO>(gate_times_up(row[i], row[I + i], act, k));
}

// ---- an RMS norm of a sublayer's OUTPUT, added to the stream ---------------------------------
// x += z / sqrt(mean(z^2) + eps) * w.  With `w_next`, the norm that reads the stream next runs on
// the new row at once: out = x / sqrt(mean(x^2) + eps_next) * w_next (the row is read where it
// was just written, by the thread that wrote it).
template <typename TO>
__global__ void __launch_bounds__(256)
rmsnorm_add_kernel(const float* __restrict__ z, const float* __restrict__ w, float eps, float* __restrict__ x,
                   const float* __restrict__ w_next, float eps_next, TO* __restrict__ out, int H) {
  __shared__ float sh[4];
  const int n = blockIdx.x;
  const float* zr = z + (size_t)n * H;
  float* xr = x + (size_t)n * H;
  float ss = 0.f;
  for (int i = threadIdx.x; i < H; i += 256) ss += zr[i] * zr[i];
  ss = block_sum<256>(ss, sh);
  const float rms = sqrtf(ss / (float)H + eps);
  float s2 = 0.f;
  for (int i = threadIdx.x; i < H; i += 256) {
    const float t = xr[i] + (zr[i] / rms) * w[i];
    xr[i] = t;
    s2 += t * t;
  }
  if (w_next == nullptr) return;
  s2 = block_sum<256>(s2, sh);
  const float rms2 = sqrtf(s2 / (float)H + eps_next);
  TO* o = out + (size_t)n * H;
  for (int i = threadIdx.x; i < H; i += 256) o[i] = from_f32<TO>((xr[i] / rms2) * w_next[i]);
}

// The same with the rows held in registers: z, x and both weights are read once, all loads issued
// before the first sum.  H % 4 == 0, H <= 1024 * IT.
template <typename TO, int IT>
__global__ void __launch_bounds__(256)
rmsnorm_add_reg_kernel(const float* __restrict__ z, const float* __restrict__ w, float eps, float* __restrict__ x,
                       const float* __restrict__ w_next, float eps_next, TO* __restrict__ out, int H) {
  __shared__ float sh[4];
  const int n = blockIdx.x;
  const float4* zr = reinterpret_cast<const float4*>(z + (size_t)n * H);
  float4* xr = reinterpret_cast<float4*>(x + (size_t)n * H);
  const float4* wr = reinterpret_cast<const float4*>(w);
  const float4* wn = reinterpret_cast<const float4*>(w_next);
  const int nv = H / 4;
  float4 a[IT], v[IT], g[IT], g2[IT];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < IT; ++i) {
    const int c = threadIdx.x + 256 * i;
    if (c < nv) {
      a[i] = zr[c];
      v[i] = xr[c];
      g[i] = wr[c];
      if (w_next) g2[i] = wn[c];
      ss += a[i].x * a[i].x + a[i].y * a[i].y + a[i].z * a[i].z + a[i].w * a[i].w;
    }
  }
  ss = block_sum<256>(ss, sh);
  const float rms = sqrtf(ss / (float)H + eps);
  float s2 = 0.f;
#pragma unroll
  for (int i = 0; i < IT; ++i) {
    const int c = threadIdx.x + 256 * i;
    if (c < nv) {
      v[i].x += (a[i].x / rms) * g[i].x;
      v[i].y += (a[i].y / rms) * g[i].y;
      v[i].z += (a[i].z / rms) * g[i].z;
      v[i].w += (a[i].w / rms) * g[i].w;
      xr[c] = v[i];
      s2 += v[i].x * v[i].x + v[i].y * v[i].y + v[i].z * v[i].z + v[i].w * v[i].w;
    }
  }
  if (w_next == nullptr) return;
  s2 = block_sum<256>(s2, sh);
  const float rms2 = sqrtf(s2 / (float)H + eps_next);
  TO* o = out + (size_t)n * H;
#pragma unroll
  for (int i = 0; i < IT; ++i) {
    const int c = threadIdx.x + 256 * i;
    if (c < nv) {
      o[4 * c + 0] = from_f32<TO>((v[i].x / rms2) * g2[i].x);
      o[4 * c + 1] = from_f32<TO>((v[i].y / rms2) * g2[i].y);
      o[4 * c + 2] = from_f32<TO>((v[i].z / rms2) * g2[i].z);
      o[4 * c + 3] = from_f32<TO>((v[i].w / rms2) * g2[i].w);
    }
  }
}

// x[n, :] += extra[n, :] (may be null) + vec[:]: what a pass over a run of layers adds at its start
__global__ void stream_entry_kernel(float* __restrict__ x, const float* __restrict__ extra,
                                    const float* __restrict__ vec, int H, size_t total) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= total) return;
  float t = x[i];
  if (extra) t += extra[i];
  x[i] = t + vec[i % H];
}

__global__ void scale_kernel(float* __restrict__ x, float s, size_t total) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < total) x[i] *= s;
}

// tokens[j] = src[idx[j]]: the ids that the sampler left on the device become the next step's
// input without a trip to the host.  An id outside the vocabulary becomes 0 (no row of the
// embedding lies there).
__global__ void take_tokens_kernel(const int* __restrict__ src, const int* __restrict__ idx, int n,
                                   int n_src, int vocab, int* __restrict__ tokens) {
  const int j = blockIdx.x * blockDim.x + threadIdx.x;
  if (j >= n) return;
  const int r = idx[j];
  const int t = (r >= 0 && r < n_src) ? src[r] : 0;
  tokens[j] = (t >= 0 && t < vocab) ? t : 0;
}

__global__ void gather_rows_kernel(const float* __restrict__ x, const int* __restrict__ idx, int H,
                                   float* __restrict__ out) {
  const int m = blockIdx.x;
  const float* s = x + (size_t)idx[m] * H;
  float* o = out + (size_t)m * H;
  for (int i = threadIdx.x; i < H; i += blockDim.x) o[i] = s[i];
}

}  // namespace tl

using namespace tl;

extern "C" {

const char* tl_last_error() { return g_err; }
int tl_page_size() { return PAGE; }      // what this library was compiled with (csrc/page.h)

int tl_embed(const void* table, int table_dt, const int* ids, int n, int H, float scale, float* out,
             hipStream_t st) {
  TL_REQUIRE(n >= 0 && H > 0, "embed: bad sizes n=%d H=%d", n, H);
  if (n == 0) return 0;
  const int nt = H >= 256 ? 256 : 64;
  if (table_dt == DT_F32)
    embed_kernel<float><<<n, nt, 0, st>>>((const float*)table, ids, H, scale, out);
  else if (table_dt == DT_BF16)
    embed_kernel<bf16><<<n, nt, 0, st>>>((const bf16*)table, ids, H, scale, out);
  else
    TL_REQUIRE(false, "embed: unknown dtype code %d", table_dt);
  TL_LAUNCH_CHECK("embed");
  return 0;
}

int tl_embed_pairs(const void* table, int table_dt, const int* ids, int n, int H, float scale, const void* pairs, long long buckets,
                   long long mul_prev, long long mul_cur, const int* row_pos, const int* row_seq, const int* cu_seqlens,
                   const int* slots, int* last, const float* w, float eps, float* out, hipStream_t st) {
  TL_REQUIRE(n >= 0 && H > 0 && table && ids && out, "embed_pairs: bad arguments n=%d H=%d", n, H);
  TL_REQUIRE(!pairs || (row_pos && row_seq && cu_seqlens && slots && last), "embed_pairs: a buffer is missing");
  TL_REQUIRE(buckets > 0 && mul_prev >= 0 && mul_cur >= 0 && mul_prev < (1LL << 31) && mul_cur < (1LL << 31),
             "embed_pairs: multipliers must lie between 0 and 2^31, buckets above 0");
  TL_REQUIRE(table_dt == DT_F32 || table_dt == DT_BF16, "embed_pairs: unknown dtype code %d", table_dt);
  if (n == 0) return 0;
  const PairTerms k{row_pos, row_seq, cu_seqlens, slots, last, buckets, mul_prev, mul_cur};
  const bool vec = H % 4 == 0 && H <= 8192 && ((uintptr_t)table | (uintptr_t)pairs | (uintptr_t)w | (uintptr_t)out) % 16 == 0;
#define TL_EP(IT)                                                                                                               \
  do {                                                                                                                          \
    if (table_dt == DT_F32)                                                                                                     \
      embed_pairs_kernel<float, IT><<<n, 256, 0, st>>>((const float*)table, ids, H, scale, (const float*)pairs, k, w, eps, out); \
    else                                                                                                                        \
      embed_pairs_kernel<bf16, IT><<<n, 256, 0, st>>>((const bf16*)table, ids, H, scale, (const bf16*)pairs, k, w, eps, out);   \
  } while (0)
  if (!vec) TL_EP(0);
  else if (H <= 1024) TL_EP(1);
  else if (H <= 2048) TL_EP(2);
  else if (H <= 4096) TL_EP(4);
  else TL_EP(8);
#undef TL_EP
  TL_LAUNCH_CHECK("embed_pairs");
  return 0;
}

int tl_rmsnorm(const float* x, const float* w, float eps, void* out, int out_dt, int n, int H,
               hipStream_t st) {
  TL_REQUIRE(n >= 0 && H > 0, "rmsnorm: bad sizes n=%d H=%d", n, H);
  if (n == 0) return 0;
  TL_REQUIRE(out_dt == DT_F32 || out_dt == DT_BF16, "rmsnorm: unknown dtype code %d", out_dt);
  const bool vec = H % 4 == 0 && H <= 8192 && ((uintptr_t)x % 16 == 0) && ((uintptr_t)w % 16 == 0);
#define TL_RMS(IT)                                                                        \
  do {                                                                                    \
    if (out_dt == DT_F32) rmsnorm_reg_kernel<float, IT><<<n, 256, 0, st>>>(x, w, eps, (float*)out, H); \
    else rmsnorm_reg_kernel<bf16, IT><<<n, 256, 0, st>>>(x, w, eps, (bf16*)out, H);        \
  } while (0)
  if (vec && H <= 1024) TL_RMS(1);
  else if (vec && H <= 2048) TL_RMS(2);
  else if (vec && H <= 4096) TL_RMS(4);
  else if (vec) TL_RMS(8);
  else if (out_dt == DT_F32)
    rmsnorm_kernel<float><<<n, 256, 0, st>>>(x, w, eps, (float*)out, H);
  else
    rmsnorm_kernel<bf16><<<n, 256, 0, st>>>(x, w, eps, (bf16*)out, H);
#undef TL_RMS
  TL_LAUNCH_CHECK("rmsnorm");
  return 0;
}

// vt (may be null): values also transposed, [nkv][d][vt_cols], row n in column
// tile_off[row_seq[n]] + row_pos[n] - 64 * (n_cached[row_seq[n]] / 64)
// x[n, H] += parts[0..n_parts)[n, H]; out = rmsnorm(x)
int tl_add_rmsnorm(float* x, const float* parts, int n_parts, const float* w, float eps, void* out, int out_dt,
                   int n, int H, hipStream_t st) {
  TL_REQUIRE(n >= 0 && H > 0 && n_parts >= 0, "add_rmsnorm: bad sizes n=%d H=%d parts=%d", n, H, n_parts);
  TL_REQUIRE(out_dt == DT_F32 || out_dt == DT_BF16, "add_rmsnorm: unknown dtype code %d", out_dt);
  TL_REQUIRE(H % 4 == 0 && H <= 8192 && ((uintptr_t)x % 16 == 0) && ((uintptr_t)w % 16 == 0) &&
             ((uintptr_t)parts % 16 == 0), "add_rmsnorm: H=%d must be a multiple of 4, at most 8192, rows 16-byte aligned", H);
  if (n == 0) return 0;
  const size_t stride = (size_t)n * H;
#define TL_ARMS(IT)                                                                                        \
  do {                                                                                                     \
    if (out_dt == DT_F32) add_rmsnorm_reg_kernel<float, IT><<<n, 256, 0, st>>>(x, parts, n_parts, stride, w, eps, (float*)out, H); \
    else add_rmsnorm_reg_kernel<bf16, IT><<<n, 256, 0, st>>>(x, parts, n_parts, stride, w, eps, (bf16*)out, H);                   \
  } while (0)
  if (H <= 1024) TL_ARMS(1);
  else if (H <= 2048) TL_ARMS(2);
  else if (H <= 4096) TL_ARMS(4);
  else TL_ARMS(8);
#undef TL_ARMS
  TL_LAUNCH_CHECK("add_rmsnorm");
  return 0;
}

// x[n, H] += parts[0..n_parts)[n, H]
int tl_add_partials(float* x, const float* parts, int n_parts, int n, int H, hipStream_t st) {
  TL_REQUIRE(n >= 0 && H > 0 && n_parts >= 0, "add_partials: bad sizes n=%d H=%d parts=%d", n, H, n_parts);
  if (n == 0 || n_parts == 0) return 0;
  const size_t total = (size_t)n * H;
  add_partials_kernel<<<(unsigned)((total + 255) / 256), 256, 0, st>>>(x, parts, n_parts, total, total);
  TL_LAUNCH_CHECK("add_partials");
  return 0;
}

// inv_freq [rotary_dim / 2], rotary_dim (even, 0..d; 0: no rotation), interleaved: see `Rotation`
int tl_rope_split(const float* qkv, const int* row_pos, const float* inv_freq, int rotary_dim, int interleaved,
                  int n, int nq, int nkv, int d, void* q, void* k, void* v, void* vt, int vt_cols,
                  const int* row_seq, const int* tile_off, const int* n_cached, int out_dt, hipStream_t st) {
  TL_REQUIRE(n >= 0 && nq > 0 && nkv >= 0 && d > 0 && d % 2 == 0,
             "rope_split: bad sizes n=%d nq=%d nkv=%d d=%d (d must be even)", n, nq, nkv, d);
  TL_REQUIRE(d <= 2 * ROPE_MAX_HALF, "rope_split: head size %d is not served (at most %d)", d, 2 * ROPE_MAX_HALF);
  TL_REQUIRE(rotary_dim >= 0 && rotary_dim <= d && rotary_dim % 2 == 0 && (rotary_dim == 0 || inv_freq != nullptr),
             "rope_split: %d rotated channels of a head of %d (even, at most the head, with their frequencies)",
             rotary_dim, d);
  const Rotation rot{inv_freq, rotary_dim, interleaved != 0};
  if (n == 0) return 0;
  if (out_dt == DT_F32)
    rope_split_kernel<float><<<n, 256, 0, st>>>(qkv, row_pos, rot, nq, nkv, d, (float*)q,
                                                 (float*)k, (float*)v, (float*)vt, vt_cols, row_seq,
                                                 tile_off, n_cached);
  else if (out_dt == DT_BF16)
    rope_split_kernel<bf16><<<n, 256, 0, st>>>(qkv, row_pos, rot, nq, nkv, d, (bf16*)q,
                                                (bf16*)k, (bf16*)v, (bf16*)vt, vt_cols, row_seq, tile_off,
                                                n_cached);
  else
    TL_REQUIRE(false, "rope_split: unknown dtype code %d", out_dt);
  TL_LAUNCH_CHECK("rope_split");
  return 0;
}

int tl_kv_commit(const void* k, const void* v, int dt, const int* row_seq, const int* row_pos,
                 const int* len_after, const int* table, int table_stride, int ring_pages, int n,
                 int nkv, int d, void* pages, hipStream_t st) {
  TL_REQUIRE(n >= 0 && nkv > 0 && d > 0 && ring_pages > 0 && table_stride > 0,
             "kv_commit: bad sizes n=%d nkv=%d d=%d ring_pages=%d table_stride=%d", n, nkv, d,
             ring_pages, table_stride);
  if (n == 0) return 0;
  const int nt = nkv * d >= 256 ? 256 : 64;
  if (dt == DT_F32)
    kv_commit_kernel<float><<<n, nt, 0, st>>>((const float*)k, (const float*)v, row_seq, row_pos,
                                               len_after, table, table_stride, ring_pages, nkv, d,
                                               (float*)pages);
  else if (dt == DT_BF16)
    kv_commit_kernel<bf16><<<n, nt, 0, st>>>((const bf16*)k, (const bf16*)v, row_seq, row_pos,
                                              len_after, table, table_stride, ring_pages, nkv, d,
                                              (bf16*)pages);
  else
    TL_REQUIRE(false, "kv_commit: unknown dtype code %d", dt);
  TL_LAUNCH_CHECK("kv_commit");
  return 0;
}

int tl_v_tiles(const float* qkv, int n, int nq, int nkv, int d, void* vt, int vt_cols, int dt, int B,
               const int* cu_seqlens, const int* tile_off, const int* n_cached, const int* len_after,
               hipStream_t st) {
  TL_REQUIRE(n >= 0 && nq >= 0 && nkv > 0 && d > 0 && B > 0, "v_tiles: bad sizes n=%d nq=%d nkv=%d d=%d B=%d", n, nq,
             nkv, d, B);
  TL_REQUIRE(vt_cols > 0 && vt_cols % PAGE == 0 && nkv <= 65535, "v_tiles: %d columns (a multiple of 64), %d KV heads",
             vt_cols, nkv);
  if (n == 0) return 0;
  const int width = (nq + 2 * nkv) * d, v_off = (nq + nkv) * d;
  const dim3 grid(vt_cols / PAGE, nkv, (d + 63) / 64);
  if (dt == DT_F32)
    v_tiles_kernel<float><<<grid, 256, 0, st>>>(qkv, width, v_off, d, (float*)vt, vt_cols, B, cu_seqlens,
                                                 tile_off, n_cached, len_after);
  else if (dt == DT_BF16)
    v_tiles_kernel<bf16><<<grid, 256, 0, st>>>(qkv, width, v_off, d, (bf16*)vt, vt_cols, B, cu_seqlens,
                                                tile_off, n_cached, len_after);
  else
    TL_REQUIRE(false, "v_tiles: unknown dtype code %d", dt);
  TL_LAUNCH_CHECK("v_tiles");
  return 0;
}

int tl_kv_commit_tiles(const void* k, const void* vt, int vt_cols, int dt, const int* row_seq, const int* row_pos,
                       int B, const int* tile_off, const int* n_cached, const int* len_after, const int* table,
                       int table_stride, int ring_pages, int n, int nkv, int d, void* pages, hipStream_t st) {
  TL_REQUIRE(n >= 0 && nkv > 0 && d > 0 && ring_pages > 0 && table_stride > 0 && B > 0,
             "kv_commit_tiles: bad sizes n=%d nkv=%d d=%d ring_pages=%d table_stride=%d B=%d", n, nkv, d,
             ring_pages, table_stride, B);
  TL_REQUIRE(vt_cols > 0 && vt_cols % PAGE == 0, "kv_commit_tiles: %d columns (a multiple of 64)", vt_cols);
  if (n == 0) return 0;
  const long long blocks = (long long)((n + 7) / 8) + (long long)(vt_cols / PAGE) * nkv;
  TL_REQUIRE(blocks < 2147483647LL, "kv_commit_tiles: too many blocks");
  if (dt == DT_F32)
    kv_commit_tiles_kernel<float><<<(unsigned)blocks, 256, 0, st>>>(
        (const float*)k, (const float*)vt, vt_cols, n, row_seq, row_pos, B, tile_off, n_cached, len_after, table,
        table_stride, ring_pages, nkv, d, (float*)pages);
  else if (dt == DT_BF16)
    kv_commit_tiles_kernel<bf16><<<(unsigned)blocks, 256, 0, st>>>(
        (const bf16*)k, (const bf16*)vt, vt_cols, n, row_seq, row_pos, B, tile_off, n_cached, len_after, table,
        table_stride, ring_pages, nkv, d, (bf16*)pages);
  else
    TL_REQUIRE(false, "kv_commit_tiles: unknown dtype code %d", dt);
  TL_LAUNCH_CHECK("kv_commit_tiles");
  return 0;
}

// tl_rope_split (q and k only) and tl_v_tiles in one launch: see rope_v_tiles_kernel
// The same from rows of values alone, v[n, nkv, d] in the type of vt (a step whose values were
// split off the projection by another kernel)
int tl_v_tiles_rows(const void* v, int n, int nkv, int d, void* vt, int vt_cols, int dt, int B,
                    const int* cu_seqlens, const int* tile_off, const int* n_cached, const int* len_after,
                    hipStream_t st) {
  TL_REQUIRE(n >= 0 && nkv > 0 && d > 0 && B > 0, "v_tiles_rows: bad sizes n=%d nkv=%d d=%d B=%d", n, nkv, d, B);
  TL_REQUIRE(vt_cols > 0 && vt_cols % PAGE == 0 && nkv <= 65535, "v_tiles_rows: %d columns (a multiple of 64), %d KV heads",
             vt_cols, nkv);
  if (n == 0) return 0;
  const dim3 grid(vt_cols / PAGE, nkv, (d + 63) / 64);
  if (dt == DT_F32)
    v_tiles_kernel<float, float><<<grid, 256, 0, st>>>((const float*)v, nkv * d, 0, d, (float*)vt, vt_cols, B, cu_seqlens,
                                                        tile_off, n_cached, len_after);
  else if (dt == DT_BF16)
    v_tiles_kernel<bf16, bf16><<<grid, 256, 0, st>>>((const bf16*)v, nkv * d, 0, d, (bf16*)vt, vt_cols, B, cu_seqlens,
                                                      tile_off, n_cached, len_after);
  else
    TL_REQUIRE(false, "v_tiles_rows: unknown dtype code %d", dt);
  TL_LAUNCH_CHECK("v_tiles_rows");
  return 0;
}

int tl_rope_v_tiles(const float* qkv, const int* row_pos, const float* inv_freq, int rotary_dim, int interleaved,
                    int n, int nq, int nkv, int d, void* q, void* k, void* vt, int vt_cols, int B,
                    const int* cu_seqlens, const int* tile_off, const int* n_cached, const int* len_after, int dt,
                    hipStream_t st) {
  TL_REQUIRE(n >= 0 && nq > 0 && nkv > 0 && d > 0 && d % 2 == 0 && d <= 2 * ROPE_MAX_HALF && B > 0,
             "rope_v_tiles: bad sizes n=%d nq=%d nkv=%d d=%d B=%d (d even, at most %d)", n, nq, nkv, d, B,
             2 * ROPE_MAX_HALF);
  TL_REQUIRE(vt_cols > 0 && vt_cols % PAGE == 0, "rope_v_tiles: %d columns are no multiple of %d", vt_cols, PAGE);
  TL_REQUIRE(rotary_dim >= 0 && rotary_dim <= d && rotary_dim % 2 == 0 && (rotary_dim == 0 || inv_freq != nullptr),
             "rope_v_tiles: %d rotated channels of a head of %d (even, at most the head, with their frequencies)",
             rotary_dim, d);
  if (n == 0) return 0;
  const Rotation rot{inv_freq, rotary_dim, interleaved != 0};
  const long long blocks = (long long)n + (long long)(vt_cols / PAGE) * nkv * ((d + 63) / 64);
  TL_REQUIRE(blocks < 2147483647LL, "rope_v_tiles: %lld workgroups are too many", blocks);
  if (dt == DT_F32)
    rope_v_tiles_kernel<float><<<(unsigned)blocks, 256, 0, st>>>(qkv, row_pos, rot, n, nq, nkv, d, (float*)q, (float*)k,
                                                                  (float*)vt, vt_cols, B, cu_seqlens, tile_off, n_cached,
                                                                  len_after);
  else if (dt == DT_BF16)
    rope_v_tiles_kernel<bf16><<<(unsigned)blocks, 256, 0, st>>>(qkv, row_pos, rot, n, nq, nkv, d, (bf16*)q, (bf16*)k,
                                                                 (bf16*)vt, vt_cols, B, cu_seqlens, tile_off, n_cached,
                                                                 len_after);
  else
    TL_REQUIRE(false, "rope_v_tiles: unknown dtype code %d", dt);
  TL_LAUNCH_CHECK("rope_v_tiles");
  return 0;
}

// n_parts >= 1: qkv is [n_parts][n][(nq + 2 nkv) d], summed on the way in
int tl_rope_commit(const float* qkv, int n_parts, const int* row_pos, const float* inv_freq, int rotary_dim,
                   int interleaved, const int* table, int table_stride, int ring_pages, int n, int nq, int nkv,
                   int d, void* q, void* pages, int dt, hipStream_t st) {
  TL_REQUIRE(n >= 0 && nq > 0 && nkv > 0 && d > 0 && d % 2 == 0 && ring_pages > 0 && table_stride > 0,
             "rope_commit: bad sizes n=%d nq=%d nkv=%d d=%d ring_pages=%d table_stride=%d", n, nq, nkv, d,
             ring_pages, table_stride);
  TL_REQUIRE(d <= 2 * ROPE_MAX_HALF, "rope_commit: head size %d is not served (at most %d)", d, 2 * ROPE_MAX_HALF);
  TL_REQUIRE(n_parts >= 1, "rope_commit: n_parts=%d", n_parts);
  TL_REQUIRE(rotary_dim >= 0 && rotary_dim <= d && rotary_dim % 2 == 0 && (rotary_dim == 0 || inv_freq != nullptr),
             "rope_commit: %d rotated channels of a head of %d (even, at most the head, with their frequencies)",
             rotary_dim, d);
  const Rotation rot{inv_freq, rotary_dim, interleaved != 0};
  if (n == 0) return 0;
  const size_t stride = (size_t)n * (nq + 2 * nkv) * d;
  const dim3 grid(n, n >= 128 ? 1 : (n >= 32 ? 4 : 8));       // few rows: cut the heads over more workgroups
  if (dt == DT_F32)
    rope_commit_kernel<float><<<grid, 256, 0, st>>>(qkv, n_parts, stride, row_pos, rot, table, table_stride,
                                                  ring_pages, nq, nkv, d, (float*)q, (float*)pages);
  else if (dt == DT_BF16)
    rope_commit_kernel<bf16><<<grid, 256, 0, st>>>(qkv, n_parts, stride, row_pos, rot, table, table_stride,
                                                 ring_pages, nq, nkv, d, (bf16*)q, (bf16*)pages);
  else
    TL_REQUIRE(false, "rope_commit: unknown dtype code %d", dt);
  TL_LAUNCH_CHECK("rope_commit");
  return 0;
}

int tl_silu_mul(const float* gu, int n, int I, void* out, int out_dt, hipStream_t st) {
  TL_REQUIRE(n >= 0 && I > 0, "silu_mul: bad sizes n=%d I=%d", n, I);
  if (n == 0) return 0;
  const int grid = n;
  if (out_dt == DT_F32)
    silu_mul_kernel<float><<<grid, 256, 0, st>>>(gu, I, (float*)out);
  else if (out_dt == DT_BF16)
    silu_mul_kernel<bf16><<<grid, 256, 0, st>>>(gu, I, (bf16*)out);
  else
    TL_REQUIRE(false, "silu_mul: unknown dtype code %d", out_dt);
  TL_LAUNCH_CHECK("silu_mul");
  return 0;
}

int tl_silu_mul_pairs(const void* gu, int n, int I, void* out, hipStream_t st) {
  TL_REQUIRE(n >= 0 && I > 0 && I % 32 == 0, "silu_mul_pairs: bad sizes n=%d I=%d (I in steps of 32)", n, I);
  TL_REQUIRE((uintptr_t)gu % 16 == 0 && (uintptr_t)out % 16 == 0, "silu_mul_pairs: buffers must be 16-byte aligned");
  if (n == 0) return 0;
  const long long chunks = (long long)n * (I / 8);
  TL_REQUIRE((chunks + 255) / 256 < 2147483647LL, "silu_mul_pairs: too many elements");
  silu_mul_pairs_kernel<<<(unsigned)((chunks + 255) / 256), 256, 0, st>>>((const bf16*)gu, chunks, I, (bf16*)out);
  TL_LAUNCH_CHECK("silu_mul_pairs");
  return 0;
}

// x null: out = layernorm(z + bias); else x += layernorm(z + bias) and out (may be null) = x
int tl_layernorm(const float* z, const float* bias, const float* w, const float* beta, float eps, float* x, void* out,
                 int out_dt, int n, int H, hipStream_t st) {
  TL_REQUIRE(n >= 0 && H > 0, "layernorm: bad sizes n=%d H=%d", n, H);
  TL_REQUIRE(x != nullptr || out != nullptr, "layernorm: nowhere to write");
  TL_REQUIRE(out == nullptr || out_dt == DT_F32 || out_dt == DT_BF16, "layernorm: unknown dtype code %d", out_dt);
  if (n == 0) return 0;
  const bool al = (uintptr_t)z % 16 == 0 && (uintptr_t)w % 16 == 0 && (uintptr_t)bias % 16 == 0 && (uintptr_t)x % 16 == 0 &&
                  (uintptr_t)beta % 16 == 0;
  const bool vec = H % 4 == 0 && H <= 8192 && al;
  const bool f32 = out == nullptr || out_dt == DT_F32;
#define TL_LN(IT)                                                                                              \
  do {                                                                                                         \
    if (f32) layernorm_reg_kernel<float, IT><<<n, 256, 0, st>>>(z, bias, w, beta, eps, x, (float*)out, H);     \
    else layernorm_reg_kernel<bf16, IT><<<n, 256, 0, st>>>(z, bias, w, beta, eps, x, (bf16*)out, H);           \
  } while (0)
  if (vec && H <= 1024) TL_LN(1);
  else if (vec && H <= 2048) TL_LN(2);
  else if (vec && H <= 4096) TL_LN(4);
  else if (vec) TL_LN(8);
  else if (f32) layernorm_kernel<float><<<n, 256, 0, st>>>(z, bias, w, beta, eps, x, (float*)out, H);
  else layernorm_kernel<bf16><<<n, 256, 0, st>>>(z, bias, w, beta, eps, x, (bf16*)out, H);
#undef TL_LN
  TL_LAUNCH_CHECK("layernorm");
  return 0;
}

int tl_cast_rows(const float* x, long long total, void* out, hipStream_t st) {
  TL_REQUIRE(total >= 0 && (total + 255) / 256 < 2147483647LL, "cast_rows: bad size %lld", total);
  if (total == 0) return 0;
  cast_rows_kernel<<<(unsigned)((total + 255) / 256), 256, 0, st>>>(x, (size_t)total, (bf16*)out);
  TL_LAUNCH_CHECK("cast_rows");
  return 0;
}

int tl_act_mul(const float* gu, int n, int I, int act, float alpha, float limit, float shift, void* out, int out_dt,
               hipStream_t st) {
  TL_REQUIRE(n >= 0 && I > 0, "act_mul: bad sizes n=%d I=%d", n, I);
  TL_REQUIRE(act == ACT_SILU || act == ACT_GELU_TANH || act == ACT_SWISH_CLAMPED || act == ACT_RELU, "act_mul: no function of code %d", act);
  TL_REQUIRE(act != ACT_SWISH_CLAMPED || limit > 0.f, "act_mul: the clamp needs a positive limit");
  if (n == 0) return 0;
  const ActConstants k{alpha, limit, shift};
  if (out_dt == DT_F32)
    act_mul_kernel<float><<<n, 256, 0, st>>>(gu, I, act, k, (float*)out);
  else if (out_dt == DT_BF16)
    act_mul_kernel<bf16><<<n, 256, 0, st>>>(gu, I, act, k, (bf16*)out);
  else
    TL_REQUIRE(false, "act_mul: unknown dtype code %d", out_dt);
  TL_LAUNCH_CHECK("act_mul");
  return 0;
}

// tl_silu_mul_pairs with the gate's function chosen (codes as tl_act_mul)
int tl_act_mul_pairs(const void* gu, int n, int I, int act, float alpha, float limit, float shift, void* out,
                     hipStream_t st) {
  TL_REQUIRE(n >= 0 && I > 0 && I % 32 == 0, "act_mul_pairs: bad sizes n=%d I=%d (I in steps of 32)", n, I);
  TL_REQUIRE(act == ACT_SILU || act == ACT_GELU_TANH || act == ACT_SWISH_CLAMPED || act == ACT_RELU, "act_mul_pairs: no function of code %d", act);
  TL_REQUIRE((uintptr_t)gu % 16 == 0 && (uintptr_t)out % 16 == 0, "act_mul_pairs: buffers must be 16-byte aligned");
  if (n == 0) return 0;
  const long long chunks = (long long)n * (I / 8);
  TL_REQUIRE((chunks + 255) / 256 < 2147483647LL, "act_mul_pairs: too many elements");
  silu_mul_pairs_kernel<<<(unsigned)((chunks + 255) / 256), 256, 0, st>>>((const bf16*)gu, chunks, I, (bf16*)out, act,
                                                                          ActConstants{alpha, limit, shift});
  TL_LAUNCH_CHECK("act_mul_pairs");
  return 0;
}

// x += rmsnorm(z; w, eps); with w_next also out = rmsnorm(x; w_next, eps_next)
int tl_rmsnorm_add(const float* z, const float* w, float eps, float* x, const float* w_next, float eps_next, void* out,
                   int out_dt, int n, int H, hipStream_t st) {
  TL_REQUIRE(n >= 0 && H > 0 && z && w && x, "rmsnorm_add: bad arguments n=%d H=%d", n, H);
  TL_REQUIRE(w_next == nullptr || (out != nullptr && (out_dt == DT_F32 || out_dt == DT_BF16)),
             "rmsnorm_add: the norm that follows needs a buffer of a known type");
  if (n == 0) return 0;
  const bool f32 = w_next == nullptr || out_dt == DT_F32;
  const bool vec = H % 4 == 0 && H <= 8192 && ((uintptr_t)z % 16 == 0) && ((uintptr_t)w % 16 == 0) &&
                   ((uintptr_t)x % 16 == 0) && ((uintptr_t)w_next % 16 == 0);
#define TL_RMSA(IT)                                                                                                  \
  do {                                                                                                               \
    if (f32) rmsnorm_add_reg_kernel<float, IT><<<n, 256, 0, st>>>(z, w, eps, x, w_next, eps_next, (float*)out, H);   \
    else rmsnorm_add_reg_kernel<bf16, IT><<<n, 256, 0, st>>>(z, w, eps, x, w_next, eps_next, (bf16*)out, H);         \
  } while (0)
  if (vec && H <= 1024) TL_RMSA(1);
  else if (vec && H <= 2048) TL_RMSA(2);
  else if (vec && H <= 4096) TL_RMSA(4);
  else if (vec) TL_RMSA(8);
  else if (f32)
    rmsnorm_add_kernel<float><<<n, 256, 0, st>>>(z, w, eps, x, w_next, eps_next, (float*)out, H);
  else
    rmsnorm_add_kernel<bf16><<<n, 256, 0, st>>>(z, w, eps, x, w_next, eps_next, (bf16*)out, H);
#undef TL_RMSA
  TL_LAUNCH_CHECK("rmsnorm_add");
  return 0;
}

// x[n, H] += extra[n, H] (may be null) + vec[H]
int tl_stream_entry(float* x, const float* extra, const float* vec, int n, int H, hipStream_t st) {
  TL_REQUIRE(n >= 0 && H > 0 && x && vec, "stream_entry: bad arguments n=%d H=%d", n, H);
  if (n == 0) return 0;
  const size_t total = (size_t)n * H;
  stream_entry_kernel<<<(unsigned)((total + 255) / 256), 256, 0, st>>>(x, extra, vec, H, total);
  TL_LAUNCH_CHECK("stream_entry");
  return 0;
}

int tl_scale(float* x, float s, long long total, hipStream_t st) {
  TL_REQUIRE(total >= 0 && x, "scale: bad arguments");
  if (total == 0) return 0;
  scale_kernel<<<(unsigned)((total + 255) / 256), 256, 0, st>>>(x, s, (size_t)total);
  TL_LAUNCH_CHECK("scale");
  return 0;
}

int tl_take_tokens(const int* src, const int* idx, int n, int n_src, int vocab, int* tokens, hipStream_t st) {
  TL_REQUIRE(n >= 0 && n_src > 0 && vocab > 0, "take_tokens: bad sizes n=%d n_src=%d vocab=%d", n, n_src, vocab);
  if (n == 0) return 0;
  take_tokens_kernel<<<(n + 255) / 256, 256, 0, st>>>(src, idx, n, n_src, vocab, tokens);
  TL_LAUNCH_CHECK("take_tokens");
  return 0;
}

int tl_gather_rows(const float* x, const int* idx, int m, int H, float* out, hipStream_t st) {
  TL_REQUIRE(m >= 0 && H > 0, "gather_rows: bad sizes m=%d H=%d", m, H);
  if (m == 0) return 0;
  gather_rows_kernel<<<m, 256, 0, st>>>(x, idx, H, out);
  TL_LAUNCH_CHECK("gather_rows");
  return 0;
}

}  // extern "C"
