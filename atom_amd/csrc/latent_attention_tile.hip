// Attention over the latent pages on the matrix cores, in tiles whose waves share all of a block's work: the form for
// the sizes that real models have (a latent of 128, 256 or 512 entries and 64 rotated ones), bfloat16, gfx950.
//
// A block of four or eight waves owns up to 16 * RT rows (token, head) of one request and one range of keys, walked 64 keys a
// chunk.  A chunk's cached rows go from their pages straight into LDS (16 bytes a lane, no registers in between), into
// one of two buffers while the other is worked on; they are staged once, row-major: the scores read them as they lie,
// the weighted sum reads them through the transposing LDS loads of gfx950.  Both products are formed transposed, so that
// a lane holds values of one row (row = lane % 16):
//
//     S^T[key][row] = K[key][:] . Q[row][:]       the waves share out (keys of the chunk) x (rows of the tile)
//     O^T[e][row]   = V^T[e][key] . P[row][key]   the waves share out the latent's entries; each takes all rows
//
// Between the two, each wave's row maxima over its keys and then the weights P (bfloat16) go through LDS.  Every wave
// keeps all rows' running maxima; a row's running sum stays in the lanes that formed its weights until the end.
//
// Three barriers a chunk: the chunk is in LDS (and the chunk before has been read) | maxima | weights.
//
// Prompt portions: every block takes all keys its tile sees.  Single tokens: a row's keys are split over `parts` blocks
// (whole chunks each), whose unnormalised results and (maximum, sum) the merge kernel joins.  Causal by absolute
// position; optional window; optional sink, a summand of the softmax's denominator without a value.
#include "lds_loads.h"

typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
typedef __attribute__((ext_vector_type(4))) short s16x4;
typedef __attribute__((ext_vector_type(2))) unsigned long u64x2;

struct LatentTileParams {
  const bf16_t* q;          // [tokens, heads, width], scaled
  const bf16_t* pages;      // [num_pages * page_size, width]
  bf16_t* out;              // [tokens, heads, rank]
  float* ws_o;              // parts > 1: [tokens, heads, parts, rank]
  float* ws_ml;             // parts > 1: [tokens, heads, parts, 2]
  const int* cu_q;          // [num_seqs + 1]
  const int* ctx_lens;      // [num_seqs]
  const int* block_tables;  // [num_seqs, max_blocks]
  const float* sink;        // [heads] or null
  int num_seqs, max_blocks, heads, page_size, window, parts, hpt, tpt;
};

constexpr int kTChunk = 64;
constexpr float kTJump = 5.5f;                // a row's running maximum moves for jumps above this; weights stay below e^5.5
constexpr int kTPPitch = kTChunk * 2 + 16;   // bytes of a row of weights in LDS

// 16-byte pieces of a staged row: the row itself and two more, so that rows at equal places fall on different banks.
// A chunk is then kTChunk * pieces of them, `pieces` loads of a whole wave.
__host__ __device__ constexpr int tile_pieces(int width) { return width / 8 + 2; }

__host__ __device__ constexpr int tile_smem(int width) {
  return 2 * kTChunk * tile_pieces(width) * 16 + 64 * kTPPitch + 4 * 64 * 4 + 2 * kTChunk * 4;
}

// Eight keys (rows 8g .. 8g + 7 of a 32-key step) of 16 entries, entry = lane % 16: the operand V^T from row-major rows.
__device__ __forceinline__ bf16x8 transposed(const unsigned char* base, int pitch) {
  typedef __attribute__((address_space(3))) s16x4 lds4;
  const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4*)base);
  const s16x4 b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds4*)(base + 4 * pitch));
  const u64x2 both = {__builtin_bit_cast(unsigned long, a), __builtin_bit_cast(unsigned long, b)};
  return __builtin_bit_cast(bf16x8, both);
}

// RANK entries of the latent, KS steps of 32 entries of a row (width = 32 KS), RT 16-row tiles of a block, NW waves.  The
// registers are counted for two waves a SIMD: the waves' Q and accumulators then all lie in ordinary registers (a wave
// with more of them keeps a part in the matrix cores' own and copies it back and forth every chunk).
template <int RANK, int KS, int RT, int NW>
__global__ void __launch_bounds__(64 * NW, 2) latent_tile_kernel(LatentTileParams p) {
  constexpr int kRank = RANK, kWidth = 32 * KS;
  constexpr int NKG = RT == 4 ? 2 : 4;   // groups of waves by keys; a group's waves share the rows
  constexpr int KT = 4 / NKG;            // 16-key tiles of a wave, in the scores
  constexpr int RS = RT / (NW / NKG);    // 16-row tiles of a wave, in the scores
  constexpr int CT = RANK / 16 / NW;     // 16-entry tiles of the latent a wave owns, in the weighted sum
  constexpr int U = tile_pieces(kWidth), kPitch = U * 16;
  extern __shared__ __attribute__((aligned(16))) unsigned char lds[];
  unsigned char* plds = lds + 2 * kTChunk * kPitch;
  float* share = reinterpret_cast<float*>(plds + 64 * kTPPitch);   // [NKG][64]: maxima, at the end sums
  int* slots = reinterpret_cast<int*>(share + 4 * 64);             // [2][64]: cache row of each key of a chunk
  const unsigned lds0 = lds_address(lds);

  const int tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(tid / kWave), lane = tid % kWave, r = lane % 16, g = lane / 16;
  // which request and which of its tokens: tiles are numbered request by request, the last ones taken first
  int b = (int)gridDim.x - 1 - (int)blockIdx.x, seq = -1, q_len = 0, q_start = 0;
  for (int s = 0; s < p.num_seqs; ++s) {
    const int ql = p.cu_q[s + 1] - p.cu_q[s];
    const int n = (ql + p.tpt - 1) / p.tpt;
    if (b < n) {
      seq = s;
      q_len = ql;
      q_start = p.cu_q[s];
      break;
    }
    b -= n;
  }
  if (seq < 0) return;
  seq = __builtin_amdgcn_readfirstlane(seq);   // the same in every lane, as is all that follows from it
  b = __builtin_amdgcn_readfirstlane(b);
  q_len = __builtin_amdgcn_readfirstlane(q_len);
  q_start = __builtin_amdgcn_readfirstlane(q_start);
  const int t0 = b * p.tpt;
  const int ctx = __builtin_amdgcn_readfirstlane(p.ctx_lens[seq]);
  const int cached = ctx - q_len;
  const int tokens_here = (q_len - t0 < p.tpt) ? q_len - t0 : p.tpt;
  const int h0 = blockIdx.y * p.hpt;
  const int first_pos = cached + t0, last_pos = first_pos + tokens_here - 1;
  const int* table = p.block_tables + (size_t)seq * p.max_blocks;
  const bool live = ctx > 0 && cached >= 0;   // a padding row has no context
  const int rows_here = tokens_here * p.hpt;  // rows of the tile that may be live; the rest are idle
  const int kg = wave % NKG, rg = wave / NKG;

  // this lane's rows in the scores
  int pos_s[RS];
  bf16x8 qreg[RS][KS];
#pragma unroll
  for (int i = 0; i < RS; ++i) {
    const int R = (rg * RS + i) * 16 + r;
    const int tt = R / p.hpt, head = h0 + R % p.hpt;
    const bool ok = live && tt < tokens_here && head < p.heads;
    pos_s[i] = ok ? first_pos + tt : -1;      // an idle row sees no key, whatever its query (a live row's, here)
    const bf16_t* src = p.q + ((size_t)(q_start + t0 + (ok ? tt : 0)) * p.heads + (ok ? head : 0)) * kWidth;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) qreg[i][ks] = *reinterpret_cast<const bf16x8*>(src + ks * 32 + g * 8);
  }

  int my_lo = 0, my_hi = 0, first_key = 0;
  if (live && last_pos >= 0) {
    first_key = (p.window > 0 && first_pos - p.window + 1 > 0) ? first_pos - p.window + 1 : 0;
    const int c_lo = first_key / kTChunk, c_hi = last_pos / kTChunk + 1;
    const int per = (c_hi - c_lo + p.parts - 1) / p.parts;
    my_lo = c_lo + (int)blockIdx.z * per;
    my_hi = my_lo + per < c_hi ? my_lo + per : c_hi;
  }
  // the last key every row sees from its first on: chunks between need no mask
  const int open_lo = (p.window > 0 && last_pos - p.window + 1 > 0) ? last_pos - p.window + 1 : 0;
  const bool whole_rows = rows_here == 16 * RT && h0 + p.hpt <= p.heads && live;

  f32x4 acc[CT][RT];
#pragma unroll
  for (int ct = 0; ct < CT; ++ct)
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) acc[ct][rt] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run[RT], l_run[RS];
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) m_run[rt] = -INFINITY;
#pragma unroll
  for (int i = 0; i < RS; ++i) l_run[i] = 0.f;

  // keys that no row of the tile sees are read as the nearest that one does
  auto readable = [&](int key) { return key > last_pos ? last_pos : key < first_key ? first_key : key; };
  auto cache_row = [&](int key) { return table[readable(key) / p.page_size] * p.page_size + readable(key) % p.page_size; };
  auto stage = [&](int buffer) {
    int row = (wave * 64 + lane) / U, col = (wave * 64 + lane) % U;
    const int* mine = slots + buffer * kTChunk;
    for (int n = wave; n < U; n += NW) {
      const int piece = col < KS * 4 ? col : 0;   // the two pieces of padding: anything that is there to read
      load_to_lds(p.pages + (size_t)mine[row] * kWidth + piece * 8, lds0 + (unsigned)(buffer * kTChunk * kPitch + n * 1024));
      row += 64 * NW / U;
      col += 64 * NW % U;
      if (col >= U) {
        col -= U;
        ++row;
      }
    }
  };

  if (my_lo < my_hi) {
    if (tid < kTChunk) {
      slots[tid] = cache_row(my_lo * kTChunk + tid);
      slots[kTChunk + tid] = cache_row((my_lo + 1) * kTChunk + tid);
    }
    __syncthreads();
    stage(0);
  }

  for (int c = my_lo; c < my_hi; ++c) {
    const int cur = (c - my_lo) & 1;
    const int kbase = c * kTChunk;
    arrived();
    lds_barrier();
    if (c + 1 < my_hi) stage(cur ^ 1);
    // the page of one key of the chunk after the next, for `slots`: asked for here, by all lanes (no branch may end
    // behind it), and first touched when everything has arrived
    const int key2 = readable((c + 2) * kTChunk + lane);
    int page2 = table[key2 / p.page_size];
    const unsigned char* klds = lds + cur * kTChunk * kPitch;

    f32x4 s[KT][RS];
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int i = 0; i < RS; ++i) s[kt][i] = f32x4{0.f, 0.f, 0.f, 0.f};
    {
      // operands are read a group of steps ahead of the products that take them
      constexpr int G = 2;
      const unsigned char* kp = klds + (kg * KT * 16 + r) * kPitch + g * 16;
      bf16x8 a[2][G][KT];
      auto read = [&](int group, bf16x8 (&to)[G][KT]) {
#pragma unroll
        for (int j = 0; j < G; ++j)
#pragma unroll
          for (int kt = 0; kt < KT; ++kt)
            to[j][kt] = *reinterpret_cast<const bf16x8*>(kp + kt * 16 * kPitch + (group * G + j) * 64);
      };
      read(0, a[0]);
#pragma unroll
      for (int group = 0; group < KS / G; ++group) {
        if (group + 1 < KS / G) read(group + 1, a[(group + 1) & 1]);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int j = 0; j < G; ++j)
#pragma unroll
          for (int kt = 0; kt < KT; ++kt)
#pragma unroll
            for (int i = 0; i < RS; ++i)
              s[kt][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[group & 1][j][kt], qreg[i][group * G + j], s[kt][i], 0, 0, 0);
        __builtin_amdgcn_sched_barrier(0);
      }
    }
    if (!(whole_rows && kbase + kTChunk - 1 <= first_pos && kbase >= open_lo)) {
#pragma unroll
      for (int kt = 0; kt < KT; ++kt)
#pragma unroll
        for (int i = 0; i < RS; ++i)
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const int key = kbase + (kg * KT + kt) * 16 + 4 * g + e;
            s[kt][i][e] = key <= pos_s[i] && (p.window <= 0 || key > pos_s[i] - p.window) ? s[kt][i][e] : -INFINITY;
          }
    }
#pragma unroll
    for (int i = 0; i < RS; ++i) {
      float mx = -INFINITY;
#pragma unroll
      for (int kt = 0; kt < KT; ++kt)
#pragma unroll
        for (int e = 0; e < 4; ++e) mx = fmaxf(mx, s[kt][i][e]);
      mx = rows_max(mx);
      if (g == 0) share[kg * 64 + (rg * RS + i) * 16 + r] = mx;
    }
    lds_barrier();
    float alpha[RT];
    bool moved = false;
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
      float m_new = m_run[rt];
#pragma unroll
      for (int k = 0; k < NKG; ++k) m_new = fmaxf(m_new, share[k * 64 + rt * 16 + r]);
      const bool jump = m_new > m_run[rt] + kTJump;   // from -inf: any key
      alpha[rt] = jump ? __expf(m_run[rt] - m_new) : 1.f;
      m_run[rt] = jump ? m_new : m_run[rt];
      moved |= jump;
    }
    if (__ballot(moved) != 0) {
#pragma unroll
      for (int ct = 0; ct < CT; ++ct)
#pragma unroll
        for (int rt = 0; rt < RT; ++rt) acc[ct][rt] *= alpha[rt];
    }
#pragma unroll
    for (int i = 0; i < RS; ++i) {
      float m = m_run[i], a = alpha[i];
#pragma unroll
      for (int k = 1; k < RT / RS; ++k)
        if (rg == k) m = m_run[k * RS + i], a = alpha[k * RS + i];
      if (m == -INFINITY) m = 0.f;   // no key seen yet: every score is -inf and every weight 0
      float sum = 0.f;
#pragma unroll
      for (int kt = 0; kt < KT; ++kt) {
        bf16x4 w;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float pr = __expf(s[kt][i][e] - m);
          sum += pr;
          w[e] = static_cast<__bf16>(pr);
        }
        *reinterpret_cast<bf16x4*>(plds + ((rg * RS + i) * 16 + r) * kTPPitch + ((kg * KT + kt) * 16 + 4 * g) * 2) = w;
      }
      l_run[i] = l_run[i] * a + sum;
    }
    lds_barrier();
    const unsigned char* vp = klds + (8 * g + r / 4) * kPitch + (wave * CT * 16 + 4 * (r % 4)) * 2;
    bf16x8 v[2];
    v[0] = transposed(vp, kPitch);
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      bf16x8 pb[RT];
#pragma unroll
      for (int rt = 0; rt < RT; ++rt)
        pb[rt] = *reinterpret_cast<const bf16x8*>(plds + (rt * 16 + r) * kTPPitch + (h * 32 + g * 8) * 2);
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        const int next = h * CT + ct + 1;
        if (next < 2 * CT) v[next & 1] = transposed(vp + (next / CT) * 32 * kPitch + (next % CT) * 32, kPitch);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int rt = 0; rt < RT; ++rt)
          acc[ct][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v[(next - 1) & 1], pb[rt], acc[ct][rt], 0, 0, 0);
        __builtin_amdgcn_sched_barrier(0);
      }
    }
    arrived();
    asm volatile("" : "+v"(page2));
    if (wave == 0) slots[cur * kTChunk + lane] = page2 * p.page_size + key2 % p.page_size;
  }

  // every row's sum: over the lanes of its wave, then over the waves that shared its keys
  lds_barrier();   // the last chunk's maxima have been read
#pragma unroll
  for (int i = 0; i < RS; ++i) {
    const float l = rows_sum(l_run[i]);
    if (g == 0) share[kg * 64 + (rg * RS + i) * 16 + r] = l;
  }
  lds_barrier();
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) {
    const int R = rt * 16 + r;
    const int tt = R / p.hpt, head = h0 + R % p.hpt;
    if (!(tt < tokens_here && head < p.heads)) continue;
    float l = 0.f;
#pragma unroll
    for (int k = 0; k < NKG; ++k) l += share[k * 64 + R];
    const size_t row_index = (size_t)(q_start + t0 + tt) * p.heads + head;
    const int e0 = wave * CT * 16 + 4 * g;
    if (p.parts == 1) {
      float denom = l, f = 1.f;
      if (p.sink) {
        const float sk = p.sink[head];
        const float top = fmaxf(m_run[rt], sk);
        f = m_run[rt] == -INFINITY ? 0.f : __expf(m_run[rt] - top);
        denom = l * f + __expf(sk - top);
      }
      const float inv = denom > 0.f ? f / denom : 0.f;
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        bf16x4 o;
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = static_cast<__bf16>(acc[ct][rt][e] * inv);
        *reinterpret_cast<bf16x4*>(p.out + row_index * kRank + e0 + ct * 16) = o;
      }
    } else {
      float* wo = p.ws_o + (row_index * p.parts + blockIdx.z) * kRank;
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) *reinterpret_cast<f32x4*>(wo + e0 + ct * 16) = acc[ct][rt];
      if (wave == 0 && g == 0) {
        float* ml = p.ws_ml + (row_index * p.parts + blockIdx.z) * 2;
        ml[0] = m_run[rt];
        ml[1] = l;
      }
    }
  }
}

static int tile_variant(int rank, int width) {
  if (rank == 128 && width == 192) return 0;
  if (rank == 256 && width == 320) return 1;
  if (rank == 512 && width == 576) return 2;
  return -1;
}

// Whether the tile kernel is built for these sizes.
ATOM_EXPORT int atom_latent_tile_supports(int rank, int width) { return tile_variant(rank, width) >= 0; }

// Without the merge of parts: the caller runs atom_latent_merge after it.
ATOM_EXPORT int atom_latent_attention_tile(const void* q, const void* pages, void* out, float* ws_o, float* ws_ml,
                                           const int* cu_q, const int* ctx_lens, const int* block_tables, int max_blocks,
                                           const float* sink, int num_seqs, int tokens, int max_q_len, int heads, int rank,
                                           int width, int page_size, int window, int parts, hipStream_t stream) {
  if (num_seqs < 0 || tokens < 0 || heads <= 0 || page_size <= 0 || max_blocks <= 0 || parts < 1) return ATOM_BAD_SHAPE;
  const int variant = tile_variant(rank, width);
  if (variant < 0) return ATOM_UNSUPPORTED;
  if (parts > 1 && (ws_o == nullptr || ws_ml == nullptr)) return ATOM_BAD_SHAPE;
  if (parts > 64) return ATOM_TOO_LARGE;
  if (tokens == 0 || num_seqs == 0) return ATOM_OK;
  // single tokens of few heads take tiles of fewer rows
  const int rt = max_q_len > 1 || heads > 32 ? 4 : heads > 16 ? 2 : 1;
  LatentTileParams p;
  p.q = (const bf16_t*)q;
  p.pages = (const bf16_t*)pages;
  p.out = (bf16_t*)out;
  p.ws_o = ws_o;
  p.ws_ml = ws_ml;
  p.cu_q = cu_q;
  p.ctx_lens = ctx_lens;
  p.block_tables = block_tables;
  p.sink = sink;
  p.num_seqs = num_seqs;
  p.max_blocks = max_blocks;
  p.heads = heads;
  p.page_size = page_size;
  p.window = window;
  p.parts = parts;
  p.hpt = heads < 16 * rt ? heads : 16 * rt;
  p.tpt = 16 * rt / p.hpt;
  const int tiles = tokens / p.tpt + num_seqs;   // at least sum over requests of ceil(q_len / tpt)
  const int chunks = (heads + p.hpt - 1) / p.hpt;
  if (chunks > 65535) return ATOM_TOO_LARGE;
  dim3 grid(tiles, chunks, parts);
#define LAUNCH(RANK, KS, RT, NW)                                                                                     \
  do {                                                                                                               \
    constexpr int smem = tile_smem(32 * KS);                                                                         \
    static_assert(smem <= 160 * 1024, "two chunks must fit in LDS");                                                 \
    static bool allowed = false;                                                                                     \
    if (!allowed) {                                                                                                  \
      if (hipFuncSetAttribute((const void*)latent_tile_kernel<RANK, KS, RT, NW>,                                     \
                              hipFuncAttributeMaxDynamicSharedMemorySize, smem) != hipSuccess)                       \
        return ATOM_LAUNCH_FAILED;                                                                                   \
      allowed = true;                                                                                                \
    }                                                                                                                \
    hipLaunchKernelGGL((latent_tile_kernel<RANK, KS, RT, NW>), grid, dim3(64 * NW), smem, stream, p);                \
  } while (0)
#define LAUNCH_ROWS(RANK, KS)                    \
  do {                                           \
    if (rt == 4) LAUNCH(RANK, KS, 4, 8);         \
    else if (rt == 2) LAUNCH(RANK, KS, 2, 8);    \
    else LAUNCH(RANK, KS, 1, 4);                 \
  } while (0)
  if (variant == 0) LAUNCH_ROWS(128, 6);
  else if (variant == 1) LAUNCH_ROWS(256, 10);
  else LAUNCH_ROWS(512, 18);
#undef LAUNCH_ROWS
#undef LAUNCH
  return launch_status();
}
