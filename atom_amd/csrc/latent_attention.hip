// Attention over a cache of latents: every token leaves one row [rank latent entries | rot rotated key entries]
// that all heads share.  A head's query is brought into the latent space first (its unrotated part times the
// head's key up-projection), so a score is one dot product of `rank + rot` entries with the cached row, and the
// weighted sum of the cached latents is expanded by the head's value up-projection afterwards:
//
//   score(t, j, h) = q_lat[t, h] . c[j] + q_rot[t, h] . k_rot[j]          (the scale is folded into q)
//   o_lat[t, h]    = sum_j softmax_j(score)[j] * c[j],   the softmax's denominator holding exp(sink[h]) as well
//
// Pages: [num_pages, page_size, rank + rot].  Three kernels:
//   latent_prepare      norms the new latents, rotates the new keys' shared part and writes both to their pages; norms
//                       the latent that queries are projected up from, where a design has one
//   heads_gemm          y[t, h, :] = alpha * x[t, h, :] W_h^T (* sigmoid(gate)), one small product per head; the
//                       absorbing product takes the rotation of the queries' rotated parts with it (QueryTurn)
//   latent_attention    scores, softmax with sink, weighted sum; any sizes, float32 or bfloat16 pages
//
//   rotation_table      the cosines and sines of a step's tokens, which every layer with the same rotation reads
//
// Rotation: entries (2i, 2i + 1) of the rotated part are a pair; its angle is position * freq[i], formed in
// float64 from a float64 table and reduced to (-pi, pi] before the float32 sine and cosine; both are multiplied
// by `mult`.
#include "common.h"

__device__ __forceinline__ void pair_angle(int position, double freq, float mult, float* c, float* s) {
  double a = (double)position * freq;
  const double two_pi = 6.283185307179586476925286766559;
  a -= two_pi * rint(a / two_pi);
  float sf, cf;
  sincosf((float)a, &sf, &cf);
  *c = cf * mult;
  *s = sf * mult;
}

// table[t][i] = (cos, sin) of token t's angle of pair i
__global__ void __launch_bounds__(256)
rotation_table_kernel(const int* __restrict__ positions, const double* __restrict__ freq, float mult, float2* __restrict__ table,
                      int tokens, int pairs) {
  const long at = (long)blockIdx.x * 256 + threadIdx.x;
  if (at >= (long)tokens * pairs) return;
  float c, s;
  pair_angle(positions[at / pairs], freq[at % pairs], mult, &c, &s);
  table[at] = make_float2(c, s);
}

ATOM_EXPORT int atom_rotation_table(const int* positions, const double* freq, float mult, void* table, int tokens, int pairs,
                                    hipStream_t stream) {
  if (tokens < 0 || pairs <= 0 || positions == nullptr || freq == nullptr || table == nullptr) return ATOM_BAD_SHAPE;
  if (tokens == 0) return ATOM_OK;
  const long blocks = ((long)tokens * pairs + 255) / 256;
  if (blocks > 0x7fffffffL / 256) return ATOM_TOO_LARGE;
  hipLaunchKernelGGL(rotation_table_kernel, dim3((unsigned)blocks), dim3(256), 0, stream, positions, freq, mult,
                     (float2*)table, tokens, pairs);
  return launch_status();
}

// proj [tokens, ld] float32 holds, where asked for, the latent of the queries at cq_off (cq_rank entries) and the
// down-projection of the keys at kv_off (rank entries, then rot).  A block a token.
template <typename T>
__global__ void __launch_bounds__(256)
latent_prepare_kernel(const float* __restrict__ proj, int ld, int cq_off, int cq_rank, const float* __restrict__ cq_w,
                      T* __restrict__ cq, int kv_off, int rank, int rot, int rot_dims, const float* __restrict__ norm_w,
                      float eps, const float2* __restrict__ turns, const int* __restrict__ slots, T* __restrict__ pages) {
  __shared__ float scratch[2][4];
  const int t = blockIdx.x;
  const int tid = threadIdx.x;
  const float* row = proj + (size_t)t * ld;
  const int slot = slots ? slots[t] : -1;   // the same for the whole block
  // both norms' sums of squares in one pass and one meeting of the waves
  float ss_q = 0.f, ss_k = 0.f;
#pragma unroll 4
  for (int i = tid; i < cq_rank; i += 256) ss_q += row[cq_off + i] * row[cq_off + i];
  if (slot >= 0) {
#pragma unroll 4
    for (int i = tid; i < rank; i += 256) ss_k += row[kv_off + i] * row[kv_off + i];
    // the shared rotated key part: by the last wave first, while the others are still adding
    T* dst = pages + (size_t)slot * (rank + rot) + rank;
    for (int i = 255 - tid; i < rot; i += 256) {
      float v = row[kv_off + rank + i];
      if (i < rot_dims) {
        const float2 cs = turns[(size_t)t * (rot_dims / 2) + (i >> 1)];
        const float other = row[kv_off + rank + (i ^ 1)];
        v = (i & 1) ? v * cs.x + other * cs.y : v * cs.x - other * cs.y;
      }
      dst[i] = from_f32<T>(v);
    }
  }
  ss_q = wave_sum(ss_q);
  ss_k = wave_sum(ss_k);
  if (tid % kWave == 0) {
    scratch[0][tid / kWave] = ss_q;
    scratch[1][tid / kWave] = ss_k;
  }
  __syncthreads();
  // x / sqrt(mean(x^2) + eps) * w
  if (cq_rank > 0) {
    const float rstd = 1.f / sqrtf((scratch[0][0] + scratch[0][1] + scratch[0][2] + scratch[0][3]) / (float)cq_rank + eps);
#pragma unroll 4
    for (int i = tid; i < cq_rank; i += 256) cq[(size_t)t * cq_rank + i] = from_f32<T>(row[cq_off + i] * rstd * cq_w[i]);
  }
  if (slot >= 0) {
    const float rstd = 1.f / sqrtf((scratch[1][0] + scratch[1][1] + scratch[1][2] + scratch[1][3]) / (float)rank + eps);
    T* dst = pages + (size_t)slot * (rank + rot);
#pragma unroll 4
    for (int i = tid; i < rank; i += 256) dst[i] = from_f32<T>(row[kv_off + i] * rstd * norm_w[i]);
  }
}

ATOM_EXPORT int atom_latent_prepare(const float* proj, int ld, int cq_off, int cq_rank, const float* cq_w, void* cq,
                                    int kv_off, int rank, int rot, int rot_dims, const float* norm_w, float eps,
                                    const void* turns, const int* slots, void* pages, int dtype, int tokens,
                                    hipStream_t stream) {
  if (tokens < 0 || ld <= 0 || cq_rank < 0 || proj == nullptr) return ATOM_BAD_SHAPE;
  if (cq_rank > 0 && (cq_off < 0 || cq_off + cq_rank > ld || cq_w == nullptr || cq == nullptr)) return ATOM_BAD_SHAPE;
  if (slots != nullptr) {
    if (rot < 0 || rank <= 0 || rot_dims < 0 || rot_dims > rot || (rot_dims & 1)) return ATOM_BAD_SHAPE;
    if (kv_off < 0 || kv_off + rank + rot > ld) return ATOM_BAD_SHAPE;
    if (norm_w == nullptr || pages == nullptr) return ATOM_BAD_SHAPE;
    if (rot_dims > 0 && turns == nullptr) return ATOM_BAD_SHAPE;
  }
  if (tokens == 0 || (cq_rank == 0 && slots == nullptr)) return ATOM_OK;
  ATOM_DISPATCH_DTYPE(dtype, hipLaunchKernelGGL((latent_prepare_kernel<T>), dim3(tokens), dim3(256), 0, stream, proj, ld,
                                                 cq_off, cq_rank, cq_w, (T*)cq, kv_off, rank, rot, rot_dims, norm_w, eps,
                                                 (const float2*)turns, slots, (T*)pages));
  return launch_status();
}

// The rotated parts of the queries, which go past the absorbing product: out[t, h, :] = scale * (x[t, h, :] with its
// first rot_dims entries turned).  The product's launch has one more column of blocks for them.
struct QueryTurn {
  const float* x;        // [tokens, ..] float32: head h's rotated part at t * ldx + h * hsx
  void* out;             // the product's output type: at t * ldo + h * hso
  long ldx, hsx, ldo, hso;
  const float2* turns;   // [tokens, rot_dims / 2]: rotation_table
  int rot, rot_dims;     // rot 0: nothing to do
  float scale;
};

// Tokens t0 .. t0 + count - 1 of head h, by a block of 256 threads: an item is a pair of neighbours (or a last single).
template <typename T>
__device__ __forceinline__ void turn_queries(const QueryTurn& q, int h, int t0, int count) {
  const int pairs = (q.rot + 1) / 2;
  for (int idx = threadIdx.x; idx < count * pairs; idx += 256) {
    const int t = t0 + idx / pairs, i = 2 * (idx % pairs);
    const float* src = q.x + (size_t)t * q.ldx + (size_t)h * q.hsx + i;
    T* dst = reinterpret_cast<T*>(q.out) + (size_t)t * q.ldo + (size_t)h * q.hso + i;
    const bool both = i + 1 < q.rot;
    float u = src[0], v = both ? src[1] : 0.f;
    if (i < q.rot_dims) {
      const float2 cs = q.turns[(size_t)t * (q.rot_dims / 2) + (i >> 1)];
      const float a = u * cs.x - v * cs.y;
      v = v * cs.x + u * cs.y;
      u = a;
    }
    dst[0] = from_f32<T>(u * q.scale);
    if (both) dst[1] = from_f32<T>(v * q.scale);
  }
}

// A gate on the product's output: y *= sigmoid(gate), one value per (token, head) or one per entry.
struct ProductGate {
  const float* g;       // null: none
  long ldg;             // entry (t, h, c) at t * ldg + h * hsg + c * csg
  int hsg, csg;
};

__device__ __forceinline__ float gate_value(const ProductGate& g, size_t t, int h, int c) {
  return 1.f / (1.f + expf(-g.g[t * g.ldg + (size_t)h * g.hsg + (size_t)c * g.csg]));
}

// ------------------------------------------------------------------ one small product per head
//
// y[t * ldy + h * hsy + n] = alpha * sum_k x[t * ldx + h * hsx + k] * w[(h * N + n) * K + k]
//                            (* sigmoid of the gate when one is given)
// float32 FMA in ascending k, 64 x 64 tiles, K walked 16 at a time through LDS.

constexpr int kHTile = 64;
constexpr int kHStep = 16;

template <typename TX, typename TW, typename TY>
__global__ void __launch_bounds__(256)
heads_gemm_kernel(const TX* __restrict__ x, long ldx, long hsx, const TW* __restrict__ w, TY* __restrict__ y, long ldy,
                  long hsy, ProductGate gate, QueryTurn turn, int m, int n, int k, float alpha) {
  __shared__ float xs[kHStep][kHTile + 4];
  __shared__ float ws[kHStep][kHTile + 4];
  const int tid = threadIdx.x;
  const int tx = tid % 16, ty = tid / 16;
  const int row0 = blockIdx.y * kHTile, col0 = blockIdx.x * kHTile;
  const int h = blockIdx.z;
  if (col0 >= n) {   // the column of blocks behind the product's
    turn_queries<TY>(turn, h, row0, m - row0 < kHTile ? m - row0 : kHTile);
    return;
  }
  const TX* xh = x + (size_t)h * hsx;
  const TW* wh = w + (size_t)h * n * k;
  float acc[4][4] = {};
  const int lrow = tid / 4;
  const int lk = (tid % 4) * 4;
  for (int k0 = 0; k0 < k; k0 += kHStep) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int kk = k0 + lk + i;
      const int xr = row0 + lrow, wr = col0 + lrow;
      xs[lk + i][lrow] = (xr < m && kk < k) ? to_f32(xh[(size_t)xr * ldx + kk]) : 0.f;
      ws[lk + i][lrow] = (wr < n && kk < k) ? to_f32(wh[(size_t)wr * k + kk]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < kHStep; ++kk) {
      float a[4], b[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) a[i] = xs[kk][ty * 4 + i];
#pragma unroll
      for (int j = 0; j < 4; ++j) b[j] = ws[kk][tx * 4 + j];
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(a[i], b[j], acc[i][j]);
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = row0 + ty * 4 + i;
    if (r >= m) continue;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = col0 + tx * 4 + j;
      if (c < n)
        y[(size_t)r * ldy + (size_t)h * hsy + c] =
            from_f32<TY>(acc[i][j] * alpha * (gate.g ? gate_value(gate, r, h, c) : 1.f));
    }
  }
}

// The same product for few rows (single tokens): a wave owns one output column of one head, reads its row of w once,
// 64 entries a step with all loads of a step independent, and multiplies it with up to 8 rows of x; the 64 partial sums
// of a row are added across the wave.  The tile kernel above walks K in steps of 16 with a barrier and a wait for
// memory in each, which for 8 rows is all it does.
constexpr int kHFewRows = 8;

template <typename TX, typename TW, typename TY>
__global__ void __launch_bounds__(256)
heads_rows_kernel(const TX* __restrict__ x, long ldx, long hsx, const TW* __restrict__ w, TY* __restrict__ y, long ldy,
                  long hsy, ProductGate gate, QueryTurn turn, int m, int n, int k, float alpha) {
  const int lane = threadIdx.x % kWave;
  const int col = blockIdx.x * (256 / kWave) + threadIdx.x / kWave;
  const int h = blockIdx.y;
  if (blockIdx.x * (256 / kWave) >= n) {   // the block behind the product's
    turn_queries<TY>(turn, h, 0, m);
    return;
  }
  if (col >= n) return;
  const TX* xh = x + (size_t)h * hsx;
  const TW* wr = w + ((size_t)h * n + col) * k;
  float acc[kHFewRows];
#pragma unroll
  for (int r = 0; r < kHFewRows; ++r) acc[r] = 0.f;
  for (int kk = lane; kk < k; kk += kWave) {
    const float wv = to_f32(wr[kk]);
#pragma unroll
    for (int r = 0; r < kHFewRows; ++r)
      if (r < m) acc[r] = fmaf(to_f32(xh[(size_t)r * ldx + kk]), wv, acc[r]);
  }
#pragma unroll
  for (int r = 0; r < kHFewRows; ++r) {
    if (r >= m) continue;
    const float total = wave_sum(acc[r]);
    if (lane == 0)
      y[(size_t)r * ldy + (size_t)h * hsy + col] =
          from_f32<TY>(total * alpha * (gate.g ? gate_value(gate, r, h, col) : 1.f));
  }
}

// The options of a per-head product from the host's plain arguments; false where they do not fit together.
static bool product_options(const float* gate, long ldg, int hsg, int csg, const float* qx, long ldqx, long hsqx, void* qout,
                            long ldqo, long hsqo, int rot, int rot_dims, const void* turns, float scale, ProductGate* g,
                            QueryTurn* q) {
  if (gate != nullptr && (ldg < 0 || hsg < 0 || csg < 0)) return false;
  *g = ProductGate{gate, ldg, hsg, csg};
  if (rot < 0 || rot_dims < 0 || rot_dims > rot || (rot_dims & 1)) return false;
  if (rot > 0 && (qx == nullptr || qout == nullptr)) return false;
  if (rot_dims > 0 && turns == nullptr) return false;
  *q = QueryTurn{qx, qout, ldqx, hsqx, ldqo, hsqo, (const float2*)turns, rot, rot_dims, scale};
  return true;
}

ATOM_EXPORT int atom_heads_gemm(const void* x, int x_dtype, long ldx, long hsx, const void* w, int w_dtype, void* y,
                                int y_dtype, long ldy, long hsy, const float* gate, long ldg, int hsg, int csg,
                                const float* qx, long ldqx, long hsqx, void* qout, long ldqo, long hsqo, int rot,
                                int rot_dims, const void* turns, float scale, int heads, int m, int n, int k, float alpha,
                                hipStream_t stream) {
  if (m < 0 || n <= 0 || k <= 0 || heads <= 0 || heads > 65535) return ATOM_BAD_SHAPE;
  if (x == nullptr || w == nullptr || y == nullptr) return ATOM_BAD_SHAPE;
  if ((unsigned)x_dtype > 1u || (unsigned)w_dtype > 1u || (unsigned)y_dtype > 1u) return ATOM_BAD_DTYPE;
  ProductGate g;
  QueryTurn q;
  if (!product_options(gate, ldg, hsg, csg, qx, ldqx, hsqx, qout, ldqo, hsqo, rot, rot_dims, turns, scale, &g, &q))
    return ATOM_BAD_SHAPE;
  if (m == 0) return ATOM_OK;
  const bool few = m <= kHFewRows;
  const int extra = rot > 0 ? 1 : 0;
  dim3 grid((n + kHTile - 1) / kHTile + extra, (m + kHTile - 1) / kHTile, heads), block(256);
  if (few) grid = dim3((n + 3) / 4 + extra, heads, 1);
  if (grid.y > 65535) return ATOM_TOO_LARGE;
#define LAUNCH(TX, TW, TY)                                                                                          \
  do {                                                                                                              \
    if (few)                                                                                                        \
      hipLaunchKernelGGL((heads_rows_kernel<TX, TW, TY>), grid, block, 0, stream, (const TX*)x, ldx, hsx, (const TW*)w, \
                         (TY*)y, ldy, hsy, g, q, m, n, k, alpha);                                                   \
    else                                                                                                            \
      hipLaunchKernelGGL((heads_gemm_kernel<TX, TW, TY>), grid, block, 0, stream, (const TX*)x, ldx, hsx, (const TW*)w, \
                         (TY*)y, ldy, hsy, g, q, m, n, k, alpha);                                                   \
  } while (0)
  switch (x_dtype * 4 + w_dtype * 2 + y_dtype) {
    case 0: LAUNCH(float, float, float); break;
    case 1: LAUNCH(float, float, bf16_t); break;
    case 2: LAUNCH(float, bf16_t, float); break;
    case 3: LAUNCH(float, bf16_t, bf16_t); break;
    case 4: LAUNCH(bf16_t, float, float); break;
    case 5: LAUNCH(bf16_t, float, bf16_t); break;
    case 6: LAUNCH(bf16_t, bf16_t, float); break;
    default: LAUNCH(bf16_t, bf16_t, bf16_t); break;
  }
#undef LAUNCH
  return launch_status();
}

// ------------------------------------------------------------------ attention over the latent pages, general form
//
// One block per (query token, head).  Keys are walked in chunks counted from position 0 with a running maximum and
// sum (float32), so a token's result depends on its own keys only: not on the batch, not on how the prompt was cut,
// not on which pages hold the keys.  The sink joins the denominator at the end.

constexpr int kLatThreads = 256;
constexpr int kLatChunk = 256;

template <typename T>
__global__ void __launch_bounds__(kLatThreads)
latent_attention_kernel(const T* __restrict__ q_abs, const T* __restrict__ pages, T* __restrict__ out,
                        const int* __restrict__ token_seq, const int* __restrict__ positions,
                        const int* __restrict__ block_tables, int max_blocks, const float* __restrict__ sink,
                        int heads, int rank, int rot, int page_size, int window) {
  extern __shared__ float smem[];
  const int width = rank + rot;
  float* qs = smem;                     // width
  float* probs = qs + width;            // kLatChunk
  float* scratch = probs + kLatChunk;   // 16
  int* rows = (int*)(scratch + 16);     // kLatChunk: the cache row of each key of the chunk
  const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int seq = token_seq[t];
  T* dst = out + ((size_t)t * heads + h) * rank;
  if (seq < 0) {
    for (int i = tid; i < rank; i += kLatThreads) dst[i] = from_f32<T>(0.f);
    return;
  }
  const int pos = positions[t];
  const int* table = block_tables + (size_t)seq * max_blocks;
  const T* qr = q_abs + ((size_t)t * heads + h) * width;
  for (int i = tid; i < width; i += kLatThreads) qs[i] = to_f32(qr[i]);
  __syncthreads();
  const int first = (window > 0 && pos - window + 1 > 0) ? pos - window + 1 : 0;
  const int last = pos;
  float acc[4] = {0.f, 0.f, 0.f, 0.f};
  float run_max = -INFINITY, run_sum = 0.f;
  const int wave = tid / kWave, lane = tid % kWave;
  for (int base = (first / kLatChunk) * kLatChunk; base <= last; base += kLatChunk) {
    const int lo = base > first ? base : first;
    const int hi = (base + kLatChunk - 1 < last) ? base + kLatChunk - 1 : last;
    const int n = hi - lo + 1;
    for (int j = tid; j < n; j += kLatThreads) {
      const int key = lo + j;
      rows[j] = table[key / page_size] * page_size + key % page_size;
    }
    __syncthreads();
    // a wave per key: lanes stride the row, so the reads are whole lines
    for (int j = wave; j < n; j += kLatThreads / kWave) {
      const T* kr = pages + (size_t)rows[j] * width;
      float s = 0.f;
      for (int i = lane; i < width; i += kWave) s += qs[i] * to_f32(kr[i]);
      s = wave_sum(s);
      if (lane == 0) probs[j] = s;
    }
    __syncthreads();
    float local_max = -INFINITY;
    for (int j = tid; j < n; j += kLatThreads) local_max = fmaxf(local_max, probs[j]);
    const float chunk_max = block_max(local_max, scratch);
    const float new_max = fmaxf(run_max, chunk_max);
    const float rescale = (run_max == -INFINITY) ? 0.f : expf(run_max - new_max);
    float local_sum = 0.f;
    for (int j = tid; j < n; j += kLatThreads) {
      const float p = expf(probs[j] - new_max);
      probs[j] = p;
      local_sum += p;
    }
    const float chunk_sum = block_sum(local_sum, scratch);
    run_sum = run_sum * rescale + chunk_sum;
    run_max = new_max;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = tid + r * kLatThreads;
      if (i < rank) {
        float a = acc[r] * rescale;
        for (int j = 0; j < n; ++j) a += probs[j] * to_f32(pages[(size_t)rows[j] * width + i]);
        acc[r] = a;
      }
    }
    __syncthreads();
  }
  // the sink: a summand of the denominator without a value
  float denom = run_sum, scale_acc = 1.f;
  if (sink) {
    const float sk = sink[h];
    const float top = fmaxf(run_max, sk);
    scale_acc = expf(run_max - top);
    denom = run_sum * scale_acc + expf(sk - top);
  }
  const float inv = scale_acc / denom;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int i = tid + r * kLatThreads;
    if (i < rank) dst[i] = from_f32<T>(acc[r] * inv);
  }
}

ATOM_EXPORT int atom_latent_attention(const void* q_abs, const void* pages, void* out, const int* token_seq,
                                      const int* positions, const int* block_tables, int max_blocks, const float* sink,
                                      int dtype, int tokens, int heads, int rank, int rot, int page_size, int window,
                                      hipStream_t stream) {
  if (tokens < 0 || heads <= 0 || rank <= 0 || rot < 0 || page_size <= 0 || max_blocks <= 0) return ATOM_BAD_SHAPE;
  if (rank > 4 * kLatThreads || heads > 65535) return ATOM_TOO_LARGE;
  if (tokens == 0) return ATOM_OK;
  const size_t smem = (size_t)(rank + rot + 2 * kLatChunk + 16) * sizeof(float);
  dim3 grid(tokens, heads), block(kLatThreads);
  ATOM_DISPATCH_DTYPE(dtype, hipLaunchKernelGGL((latent_attention_kernel<T>), grid, block, smem, stream, (const T*)q_abs,
                                                 (const T*)pages, (T*)out, token_seq, positions, block_tables, max_blocks,
                                                 sink, heads, rank, rot, page_size, window));
  return launch_status();
}

// ------------------------------------------------------------------ the per-head products on the matrix cores
//
// The same product as heads_gemm with bfloat16 weights: the head's weight rows are the A operand and the tokens the B
// operand, both read straight from memory (a float32 input is rounded to bfloat16 on the way, or, where the product is
// to be the float32 one, split into three bfloat16 pieces that are multiplied one by one), so a lane ends up with four
// consecutive columns of one token.  Three kernels: the exact one (a block of 2 x 2 waves owns 64 tokens x 64 columns),
// one for many rows and one for few.  All need k % 8 == 0 and offsets and strides of x that keep its 8-element pieces
// aligned.

typedef __attribute__((ext_vector_type(4))) float hg_f32x4;
typedef __attribute__((ext_vector_type(8))) __bf16 hg_bf16x8;

__device__ __forceinline__ hg_bf16x8 hg_load8(const bf16_t* p, bool ok) {
  const hg_bf16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  return ok ? *reinterpret_cast<const hg_bf16x8*>(p) : zero;
}

// A float32 input in three bfloat16 pieces, x = hi + mid + lo exactly (3 x 8 bits of mantissa): the products of each
// piece with a bfloat16 weight are exact in float32 and the matrix cores add them in float32, so the three products
// together are the float32 product, at three matrix instructions instead of 32 multiply-adds a lane.
__device__ __forceinline__ void hg_load8_split(const float* p, bool ok, hg_bf16x8* hi, hg_bf16x8* mid, hg_bf16x8* lo) {
  const hg_bf16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  *hi = *mid = *lo = zero;
  if (ok) {
    const hg_f32x4 a = *reinterpret_cast<const hg_f32x4*>(p), b = *reinterpret_cast<const hg_f32x4*>(p + 4);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const float v = i < 4 ? a[i] : b[i - 4];
      const __bf16 h = static_cast<__bf16>(v);
      const float r1 = v - static_cast<float>(h);
      const __bf16 m = static_cast<__bf16>(r1);
      const float r2 = r1 - static_cast<float>(m);
      (*hi)[i] = h;
      (*mid)[i] = m;
      (*lo)[i] = static_cast<__bf16>(r2);
    }
  }
}

template <typename TY>
__global__ void __launch_bounds__(256)
heads_gemm_split_kernel(const float* __restrict__ x, long ldx, long hsx, const bf16_t* __restrict__ w, TY* __restrict__ y,
                       long ldy, long hsy, ProductGate gate, QueryTurn turn, int m, int n, int k, float alpha) {
  const int tid = threadIdx.x, wave = tid / kWave, lane = tid % kWave, r = lane % 16, g = lane / 16;
  const int h = blockIdx.z;
  if (blockIdx.x * 64 >= n) {   // the column of blocks behind the product's
    turn_queries<TY>(turn, h, blockIdx.y * 64, m - (int)blockIdx.y * 64 < 64 ? m - (int)blockIdx.y * 64 : 64);
    return;
  }
  const int row0 = blockIdx.y * 64 + (wave / 2) * 32;
  const int col0 = blockIdx.x * 64 + (wave % 2) * 32;
  const float* xrow[2];
  bool rok[2];
#pragma unroll
  for (int rt = 0; rt < 2; ++rt) {
    const int row = row0 + rt * 16 + r;
    rok[rt] = row < m;
    xrow[rt] = x + (size_t)(rok[rt] ? row : 0) * ldx + (size_t)h * hsx;
  }
  const bf16_t* wrow[2];
  bool cok[2];
#pragma unroll
  for (int ct = 0; ct < 2; ++ct) {
    const int col = col0 + ct * 16 + r;
    cok[ct] = col < n;
    wrow[ct] = w + ((size_t)h * n + (cok[ct] ? col : 0)) * k;
  }
  hg_f32x4 acc[2][2];
#pragma unroll
  for (int ct = 0; ct < 2; ++ct)
#pragma unroll
    for (int rt = 0; rt < 2; ++rt) acc[ct][rt] = hg_f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < k; k0 += 32) {
    const int kk = k0 + 8 * g;
    const bool kok = kk < k;
    hg_bf16x8 xb[2], xm[2], xl[2], wa[2];
#pragma unroll
    for (int rt = 0; rt < 2; ++rt) hg_load8_split(xrow[rt] + kk, kok && rok[rt], &xb[rt], &xm[rt], &xl[rt]);
#pragma unroll
    for (int ct = 0; ct < 2; ++ct) wa[ct] = hg_load8(wrow[ct] + kk, kok && cok[ct]);
#pragma unroll
    for (int ct = 0; ct < 2; ++ct)
#pragma unroll
      for (int rt = 0; rt < 2; ++rt) {
        // the small pieces first
        acc[ct][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wa[ct], xl[rt], acc[ct][rt], 0, 0, 0);
        acc[ct][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wa[ct], xm[rt], acc[ct][rt], 0, 0, 0);
        acc[ct][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wa[ct], xb[rt], acc[ct][rt], 0, 0, 0);
      }
  }
#pragma unroll
  for (int rt = 0; rt < 2; ++rt) {
    const int row = row0 + rt * 16 + r;
    if (row >= m) continue;
#pragma unroll
    for (int ct = 0; ct < 2; ++ct) {
      const int col = col0 + ct * 16 + 4 * g;
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (col + i < n)
          y[(size_t)row * ldy + (size_t)h * hsy + col + i] =
              from_f32<TY>(acc[ct][rt][i] * alpha * (gate.g ? gate_value(gate, row, h, col + i) : 1.f));
    }
  }
}

// For many rows: a block of 2 x 2 waves owns 64 tokens x 128 columns, a wave 32 x 64 of them; K is walked 64 at a time
// (whole lines of bfloat16 rows), the next 64's pieces asked for before this step's products.  `vec`: y, its strides and the
// gate's suit eight columns at a time (n % 8 = 0).
constexpr int kHWideTokens = 64;

template <typename TX>
struct HeadPieces;
template <>
struct HeadPieces<bf16_t> {
  hg_bf16x8 v;
  __device__ __forceinline__ void load(const bf16_t* p) { v = *reinterpret_cast<const hg_bf16x8*>(p); }
  __device__ __forceinline__ hg_bf16x8 get(bool ok) const {
    const hg_bf16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
    return ok ? v : zero;
  }
};
template <>
struct HeadPieces<float> {
  hg_f32x4 a, b;
  __device__ __forceinline__ void load(const float* p) {
    a = *reinterpret_cast<const hg_f32x4*>(p);
    b = *reinterpret_cast<const hg_f32x4*>(p + 4);
  }
  __device__ __forceinline__ hg_bf16x8 get(bool ok) const {
    hg_bf16x8 out;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      out[i] = static_cast<__bf16>(ok ? a[i] : 0.f);
      out[4 + i] = static_cast<__bf16>(ok ? b[i] : 0.f);
    }
    return out;
  }
};

template <typename TX, typename TY>
__global__ void __launch_bounds__(256, 2)
heads_gemm_wide_kernel(const TX* __restrict__ x, long ldx, long hsx, const bf16_t* __restrict__ w, TY* __restrict__ y,
                       long ldy, long hsy, ProductGate gate, QueryTurn turn, int m, int n, int k, float alpha, int vec) {
  const int tid = threadIdx.x, wave = tid / kWave, lane = tid % kWave, r = lane % 16, g = lane / 16;
  const int h = blockIdx.z;
  if ((int)blockIdx.x * 128 >= n) {   // the column of blocks behind the product's
    const int t0 = (int)blockIdx.y * kHWideTokens;
    turn_queries<TY>(turn, h, t0, m - t0 < kHWideTokens ? m - t0 : kHWideTokens);
    return;
  }
  constexpr int RT = kHWideTokens / 32, CT = 4;   // 16-row and 16-column tiles of a wave
  const int row0 = blockIdx.y * kHWideTokens + (wave / 2) * (RT * 16);
  const int col0 = blockIdx.x * 128 + (wave % 2) * 64;
  // rows and columns beyond the product's are read as its last ones and not written
  const TX* xrow[RT];
  const bf16_t* wrow[CT];
#pragma unroll
  for (int j = 0; j < RT; ++j)
    xrow[j] = x + (size_t)(row0 + j * 16 + r < m ? row0 + j * 16 + r : m - 1) * ldx + (size_t)h * hsx;
#pragma unroll
  for (int i = 0; i < CT; ++i)
    wrow[i] = w + ((size_t)h * n + (col0 + i * 16 + r < n ? col0 + i * 16 + r : n - 1)) * k;
  hg_f32x4 acc[CT][RT];
#pragma unroll
  for (int i = 0; i < CT; ++i)
#pragma unroll
    for (int j = 0; j < RT; ++j) acc[i][j] = hg_f32x4{0.f, 0.f, 0.f, 0.f};
  HeadPieces<TX> xp[2][2][RT];
  HeadPieces<bf16_t> wp[2][2][CT];
  auto fetch = [&](int buffer, int k0) {
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const int at = k0 + s * 32 + 8 * g, kk = at < k ? at : k - 8;   // past the end: the last piece, counted as zeros
#pragma unroll
      for (int j = 0; j < RT; ++j) xp[buffer][s][j].load(xrow[j] + kk);
#pragma unroll
      for (int i = 0; i < CT; ++i) wp[buffer][s][i].load(wrow[i] + kk);
    }
  };
  auto multiply = [&](int buffer, int k0) {
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const bool ok = k0 + s * 32 + 8 * g < k;
      hg_bf16x8 xb[RT];
#pragma unroll
      for (int j = 0; j < RT; ++j) xb[j] = xp[buffer][s][j].get(ok);
#pragma unroll
      for (int i = 0; i < CT; ++i)
#pragma unroll
        for (int j = 0; j < RT; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wp[buffer][s][i].get(true), xb[j], acc[i][j], 0, 0, 0);
    }
  };
  fetch(0, 0);
  if (k <= 128) {   // nothing behind the second fetch: no third one that would only be thrown away
    fetch(1, 64);
    multiply(0, 0);
    multiply(1, 64);
  } else {
    for (int k0 = 0; k0 < k; k0 += 128) {
      fetch(1, k0 + 64);
      __builtin_amdgcn_sched_barrier(0);
      multiply(0, k0);
      fetch(0, k0 + 128);
      __builtin_amdgcn_sched_barrier(0);
      multiply(1, k0 + 64);
    }
  }
  // lane (r, g) holds columns col0 + 16 i + 4g .. + 3 of row row0 + 16 j + r; through LDS, so that whole lines are written
  __shared__ __attribute__((aligned(16))) float tile[kHWideTokens][128 + 4];
#pragma unroll
  for (int j = 0; j < RT; ++j)
#pragma unroll
    for (int i = 0; i < CT; ++i)
      *reinterpret_cast<hg_f32x4*>(&tile[(wave / 2) * (RT * 16) + j * 16 + r][(wave % 2) * 64 + i * 16 + 4 * g]) = acc[i][j] * alpha;
  __syncthreads();
  const int c = (tid % 16) * 8, col = blockIdx.x * 128 + c;
  for (int t = tid / 16; t < kHWideTokens; t += 16) {
    const int row = (int)blockIdx.y * kHWideTokens + t;
    if (row >= m || col >= n) break;
    float v[8];
#pragma unroll
    for (int q = 0; q < 8; ++q) v[q] = tile[t][c + q];
    TY* dst = y + (size_t)row * ldy + (size_t)h * hsy + col;
    if (vec) {
      if (gate.g && gate.csg) {
        const float* gp = gate.g + row * gate.ldg + (size_t)h * gate.hsg + col;
        const hg_f32x4 ga = *reinterpret_cast<const hg_f32x4*>(gp), gb = *reinterpret_cast<const hg_f32x4*>(gp + 4);
#pragma unroll
        for (int q = 0; q < 8; ++q) v[q] *= 1.f / (1.f + expf(-(q < 4 ? ga[q] : gb[q - 4])));
      } else if (gate.g) {
        const float f = gate_value(gate, row, h, 0);
#pragma unroll
        for (int q = 0; q < 8; ++q) v[q] *= f;
      }
      if constexpr (sizeof(TY) == 2) {
        hg_bf16x8 o;
#pragma unroll
        for (int q = 0; q < 8; ++q) o[q] = static_cast<__bf16>(v[q]);
        *reinterpret_cast<hg_bf16x8*>(dst) = o;
      } else {
        *reinterpret_cast<hg_f32x4*>(dst) = hg_f32x4{v[0], v[1], v[2], v[3]};
        *reinterpret_cast<hg_f32x4*>(dst + 4) = hg_f32x4{v[4], v[5], v[6], v[7]};
      }
    } else {
#pragma unroll
      for (int q = 0; q < 8; ++q)
        if (col + q < n) dst[q] = from_f32<TY>(v[q] * (gate.g ? gate_value(gate, row, h, col + q) : 1.f));
    }
  }
}

constexpr int kHWideRows = 96;   // from here on the wide tiles

// For fewer rows: a block owns 16 columns of one head and 16 tokens; its four waves share out K (wave v the steps v, v + 4,
// ..., four of them in flight) and meet once to add their sums, in the order of the waves.
template <typename TX, typename TY>
__global__ void __launch_bounds__(256)
heads_gemm_few_kernel(const TX* __restrict__ x, long ldx, long hsx, const bf16_t* __restrict__ w, TY* __restrict__ y,
                      long ldy, long hsy, ProductGate gate, QueryTurn turn, int m, int n, int k, float alpha) {
  __shared__ float part[4][16][17];
  const int tid = threadIdx.x, wave = tid / kWave, lane = tid % kWave, r = lane % 16, g = lane / 16;
  const int h = blockIdx.z, row0 = blockIdx.y * 16, col0 = blockIdx.x * 16;
  if (col0 >= n) {   // the column of blocks behind the product's
    turn_queries<TY>(turn, h, row0, m - row0 < 16 ? m - row0 : 16);
    return;
  }
  const TX* xr = x + (size_t)(row0 + r < m ? row0 + r : m - 1) * ldx + (size_t)h * hsx;
  const bf16_t* wr = w + ((size_t)h * n + (col0 + r < n ? col0 + r : n - 1)) * k;
  hg_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = wave * 32; k0 < k; k0 += 512) {
    HeadPieces<TX> xp[4];
    HeadPieces<bf16_t> wp[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int at = k0 + i * 128 + 8 * g, kk = at < k ? at : k - 8;   // past the end: the last piece, counted as zeros
      xp[i].load(xr + kk);
      wp[i].load(wr + kk);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wp[i].get(true), xp[i].get(k0 + i * 128 + 8 * g < k), acc, 0, 0, 0);
  }
  // lane (r, g) holds columns 4g .. 4g + 3 of row r
#pragma unroll
  for (int i = 0; i < 4; ++i) part[wave][r][4 * g + i] = acc[i];
  __syncthreads();
  const int row = row0 + tid / 16, col = col0 + tid % 16;
  if (row >= m || col >= n) return;
  float v = part[0][tid / 16][tid % 16];
#pragma unroll
  for (int i = 1; i < 4; ++i) v += part[i][tid / 16][tid % 16];
  v *= alpha * (gate.g ? gate_value(gate, row, h, col) : 1.f);
  y[(size_t)row * ldy + (size_t)h * hsy + col] = from_f32<TY>(v);
}

ATOM_EXPORT int atom_heads_gemm_mfma_supports(int x_dtype, int w_dtype, long x_offset, long ldx, long hsx, int k) {
  if (w_dtype != ATOM_BF16 || k % 8) return 0;
  const long unit = x_dtype == ATOM_BF16 ? 8 : 4;   // elements of 16 bytes
  return x_offset % unit == 0 && ldx % unit == 0 && hsx % unit == 0;
}

ATOM_EXPORT int atom_heads_gemm_mfma(const void* x, int x_dtype, long ldx, long hsx, const void* w, void* y, int y_dtype,
                                     long ldy, long hsy, const float* gate, long ldg, int hsg, int csg, const float* qx,
                                     long ldqx, long hsqx, void* qout, long ldqo, long hsqo, int rot, int rot_dims,
                                     const void* turns, float scale, int heads, int m, int n, int k, float alpha, int split,
                                     hipStream_t stream) {
  if (m < 0 || n <= 0 || k <= 0 || heads <= 0 || heads > 65535 || (k % 8)) return ATOM_BAD_SHAPE;
  if (split && x_dtype != ATOM_F32) return ATOM_UNSUPPORTED;   // only a float32 input has pieces to split into
  if (x == nullptr || w == nullptr || y == nullptr) return ATOM_BAD_SHAPE;
  if ((unsigned)x_dtype > 1u || (unsigned)y_dtype > 1u) return ATOM_BAD_DTYPE;
  ProductGate g;
  QueryTurn q;
  if (!product_options(gate, ldg, hsg, csg, qx, ldqx, hsqx, qout, ldqo, hsqo, rot, rot_dims, turns, scale, &g, &q))
    return ATOM_BAD_SHAPE;
  if (m == 0) return ATOM_OK;
  dim3 grid((n + 63) / 64 + (rot > 0 ? 1 : 0), (m + 63) / 64, heads), block(256);
  if (grid.y > 65535) return ATOM_TOO_LARGE;
  if (!split && m >= kHWideRows) {
    const long unit = 8;   // entries that are read or written together
    const int vec = n % unit == 0 && ldy % unit == 0 && hsy % unit == 0 && (size_t)y % 16 == 0 &&
                    (g.g == nullptr || g.csg == 0 || ((size_t)g.g % 16 == 0 && g.ldg % 4 == 0 && g.hsg % 4 == 0));
    grid = dim3((n + 127) / 128 + (rot > 0 ? 1 : 0), (m + kHWideTokens - 1) / kHWideTokens, heads);
#define WIDE(TX, TY)                                                                                                \
  hipLaunchKernelGGL((heads_gemm_wide_kernel<TX, TY>), grid, block, 0, stream, (const TX*)x, ldx, hsx, (const bf16_t*)w, \
                     (TY*)y, ldy, hsy, g, q, m, n, k, alpha, vec)
    switch (x_dtype * 2 + y_dtype) {
      case 0: WIDE(float, float); break;
      case 1: WIDE(float, bf16_t); break;
      case 2: WIDE(bf16_t, float); break;
      default: WIDE(bf16_t, bf16_t); break;
    }
#undef WIDE
    return launch_status();
  }
  if (!split) {
    grid = dim3((n + 15) / 16 + (rot > 0 ? 1 : 0), (m + 15) / 16, heads);
#define FEW(TX, TY)                                                                                                 \
  hipLaunchKernelGGL((heads_gemm_few_kernel<TX, TY>), grid, block, 0, stream, (const TX*)x, ldx, hsx, (const bf16_t*)w, \
                     (TY*)y, ldy, hsy, g, q, m, n, k, alpha)
    switch (x_dtype * 2 + y_dtype) {
      case 0: FEW(float, float); break;
      case 1: FEW(float, bf16_t); break;
      case 2: FEW(bf16_t, float); break;
      default: FEW(bf16_t, bf16_t); break;
    }
#undef FEW
    return launch_status();
  }
  if (y_dtype == ATOM_F32)
    hipLaunchKernelGGL((heads_gemm_split_kernel<float>), grid, block, 0, stream, (const float*)x, ldx, hsx, (const bf16_t*)w,
                       (float*)y, ldy, hsy, g, q, m, n, k, alpha);
  else
    hipLaunchKernelGGL((heads_gemm_split_kernel<bf16_t>), grid, block, 0, stream, (const float*)x, ldx, hsx,
                       (const bf16_t*)w, (bf16_t*)y, ldy, hsy, g, q, m, n, k, alpha);
  return launch_status();
}
