// Latent attention: queries through a low-rank latent, keys and values as linear maps of ONE cached
// latent row per token (c, kv_rank wide) plus one rotated key part shared by all heads, causal or
// limited to a sliding window:
//   score[h, s] = (q[h, :dim] . (Wuk_h c_s) + q[h, dim:] . r_s) * scale,   out[h] = sum_s p_s Wuv_h c_s
//
//   prepare   from the down projections' output: RMS-normed query latent, RMS-normed latent row and rotated
//             key part into the caches, cosines / sines of the token for the queries' rotation
//   decode    (few tokens) the maps are moved to the query side: q' = Wuk_h^T q (absorb), attention over
//             the latent rows themselves -- all heads share them, 16 heads are the columns of the matrix
//             instructions -- and Wuv_h applied to the result (output, which merges the splits of the
//             key range). The cache is read once per 16 heads.
//   prefill   (prompts) keys and values of the visible rows come from one matrix product over the latent
//             rows (the library's linear), then a causal / windowed flash kernel: 32 queries per wave,
//             64 keys per step; no score ever leaves the registers.
//   plain     one workgroup per query and head: fp32 models, sizes the others do not cover.
//
// Positions: a token's slot in the cache minus its row's first slot (left-padded batches). Angles are
// formed and reduced in double precision and rounded to fp32 once: no table, no longest sequence.
#include "hybrid.cuh"

namespace mui {

struct LatentParams {
  const void* down;      // [tokens, down_pitch]: query latent | kv latent | key rotation part (last two: if kv)
  long down_pitch;
  const void* q_gain;    // [q_rank]
  const void* kv_gain;   // [kv_rank] or null: no kv rows here (they are another layer's)
  float eps;
  const double* inv_freq;  // [rot / 2]
  void* q_latent;          // [tokens, q_rank]
  float* cos_sin;          // [tokens, rot]: cos | sin
  int q_rank;

  const void* q;  // [tokens, heads * (dim + rot)], not rotated
  const void *w_uk, *w_uv;  // [heads * dim, kv_rank], [heads * vdim, kv_rank]
  void *c_cache, *r_cache;  // rows of kv_rank / rot elements, batch strides below
  long c_batch, r_batch;
  const int64_t* cache_position;  // [t]: slot of token t (the same for every batch row)
  const int64_t* row_start;       // [batch] first slot of the row, or null (0)
  int batch, t, heads, dim, rot, vdim, kv_rank, window, max_cache_len;
  float scale;
  void* out;  // [tokens, heads * vdim]

  void* q_abs;       // decode: [tokens, heads, kp] 16-bit
  float* part;       // decode: [tokens, heads, splits, kv_rank]
  float* part_ml;    // decode: [tokens, heads, splits, 2]: running maximum, sum
  int kp, splits, split_keys;

  const void* kv;    // prefill: [keys, heads * (dim + vdim)], key row 0 = slot kv_first
  int kv_first, kv_rows, q_first, b0;
};

// ---------------------------------------------------------------------------------------
// prepare: one workgroup per token
// ---------------------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256) latent_prepare_kernel(const LatentParams p) {
  typedef typename T::storage S;
  __shared__ float red[2][4];
  const int tok = blockIdx.x, b = tok / p.t, t = threadIdx.x;
  const S* row = (const S*)p.down + (long)tok * p.down_pitch;
  const S* cr = row + p.q_rank;
  const bool kv_here = p.kv_gain != nullptr;
  const long slot = p.cache_position[tok - b * p.t];
  const long pos = slot - (p.row_start ? p.row_start[b] : 0);
  float sq = 0.f, sk = 0.f;
#pragma unroll 4
  for (int i = t; i < p.q_rank; i += 256) {
    const float v = T::one(row[i]);
    sq = fmaf(v, v, sq);
  }
  if (kv_here) {
#pragma unroll 4
    for (int i = t; i < p.kv_rank; i += 256) {
      const float v = T::one(cr[i]);
      sk = fmaf(v, v, sk);
    }
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((t & 63) == 0) {
    red[0][t >> 6] = sq;
    red[1][t >> 6] = sk;
  }
  const bool kv = kv_here && slot >= 0 && slot < p.max_cache_len;
  const int half = p.rot >> 1;
  const S* kr = cr + p.kv_rank;
  for (int i = t; i < half; i += 256) {
    float c, s;
    rope_angle((double)(pos > 0 ? pos : 0), p.inv_freq[i], c, s);
    p.cos_sin[(long)tok * p.rot + i] = c;
    p.cos_sin[(long)tok * p.rot + half + i] = s;
    if (kv) {
      S* dst = (S*)p.r_cache + b * p.r_batch + slot * p.rot;
      const float u = T::one(kr[i]), v = T::one(kr[half + i]);
      dst[i] = T::pack(u * c - v * s);
      dst[half + i] = T::pack(v * c + u * s);
    }
  }
  __syncthreads();
  float rs = rsqrtf(((red[0][0] + red[0][1]) + (red[0][2] + red[0][3])) / (float)p.q_rank + p.eps);
  S* ql = (S*)p.q_latent + (long)tok * p.q_rank;
#pragma unroll 4
  for (int i = t; i < p.q_rank; i += 256) ql[i] = T::pack(T::one(((const S*)p.q_gain)[i]) * (T::one(row[i]) * rs));
  if (!kv) return;
  rs = rsqrtf(((red[1][0] + red[1][1]) + (red[1][2] + red[1][3])) / (float)p.kv_rank + p.eps);
  S* dst = (S*)p.c_cache + b * p.c_batch + slot * p.kv_rank;
#pragma unroll 4
  for (int i = t; i < p.kv_rank; i += 256) dst[i] = T::pack(T::one(((const S*)p.kv_gain)[i]) * (T::one(cr[i]) * rs));
}

// element e of a head's query (dim unrotated, then rot rotated)
template <typename T>
__device__ __forceinline__ float rotated_q(const typename T::storage* qh, const float* cs, int dim, int rot, int e) {
  if (e < dim) return T::one(qh[e]);
  const int j = e - dim, half = rot >> 1;
  const int i = j < half ? j : j - half;
  const float u = T::one(qh[dim + i]), v = T::one(qh[dim + half + i]);
  const float c = cs[i], s = cs[half + i];
  return j < half ? u * c - v * s : v * c + u * s;
}

// elements e0 .. e0 + 7 of the same, rounded and packed; vec: dim a multiple of 8 and rot of 16, whole chunks by
// 128-bit loads
template <typename T>
__device__ __forceinline__ u32x4 rotated_q8(const uint16_t* qh, const float* cs, int dim, int rot, int e0, bool vec) {
  const u32x4 zero = {0u, 0u, 0u, 0u};
  if (vec) {
    if (e0 < dim) return ld16(qh + e0);
    if (e0 >= dim + rot) return zero;
    const int half = rot >> 1, j = e0 - dim, i = j < half ? j : j - half;
    float u[8], v[8], c[8], s[8], o[8];
    unpack8<T>(ld16(qh + dim + i), u);
    unpack8<T>(ld16(qh + dim + half + i), v);
    load8<F32>(cs + i, c);
    load8<F32>(cs + half + i, s);
#pragma unroll
    for (int k = 0; k < 8; ++k) o[k] = j < half ? u[k] * c[k] - v[k] * s[k] : v[k] * c[k] + u[k] * s[k];
    return pack8<T>(o);
  }
  uint32_t w[8];
#pragma unroll
  for (int k = 0; k < 8; ++k)
    w[k] = e0 + k < dim + rot ? T::pack(rotated_q<T>(qh, cs, dim, rot, e0 + k)) : (uint16_t)0;
  return u32x4{w[0] | (w[1] << 16), w[2] | (w[3] << 16), w[4] | (w[5] << 16), w[6] | (w[7] << 16)};
}

// first and last visible slot of token tok (of batch row b)
__device__ __forceinline__ void visible(const LatentParams& p, int tok, int b, long& lo, long& hi) {
  hi = p.cache_position[tok - b * p.t];
  hi = hi < p.max_cache_len ? hi : p.max_cache_len - 1;
  lo = p.window > 0 ? hi - p.window + 1 : 0;
  const long first = p.row_start ? p.row_start[b] : 0;
  lo = lo > first ? lo : first;
  lo = lo > 0 ? lo : 0;
}

extern __shared__ __align__(16) unsigned char la_smem[];

// ---------------------------------------------------------------------------------------
// plain: grid (heads, tokens)
// ---------------------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256) latent_plain_kernel(const LatentParams p) {
  typedef typename T::storage S;
  __shared__ float red[4];
  float* q = (float*)la_smem;          // dim + rot
  float* qa = q + p.dim + p.rot;       // kv_rank
  float* o = qa + p.kv_rank;           // kv_rank
  float* pr = o + p.kv_rank;           // 256
  const int h = blockIdx.x, tok = blockIdx.y, b = tok / p.t, t = threadIdx.x;
  const int hd = p.dim + p.rot;
  const S* qh = (const S*)p.q + ((long)tok * p.heads + h) * hd;
  const float* cs = p.cos_sin + (long)tok * p.rot;
  for (int i = t; i < hd; i += 256) q[i] = rotated_q<T>(qh, cs, p.dim, p.rot, i);
  __syncthreads();
  const S* wk = (const S*)p.w_uk + (long)h * p.dim * p.kv_rank;
  for (int r = t; r < p.kv_rank; r += 256) {
    float a = 0.f;
    for (int d = 0; d < p.dim; ++d) a = fmaf(q[d], T::one(wk[(long)d * p.kv_rank + r]), a);
    qa[r] = a;
    o[r] = 0.f;
  }
  __syncthreads();
  long lo, hi;
  visible(p, tok, b, lo, hi);
  const S* cc = (const S*)p.c_cache + b * p.c_batch;
  const S* rc = (const S*)p.r_cache + b * p.r_batch;
  float m = -1e30f, l = 0.f;
  for (long s0 = lo; s0 <= hi; s0 += 256) {
    const long s = s0 + t;
    float sc = -INFINITY;
    if (s <= hi) {
      float a = 0.f;
      for (int r = 0; r < p.kv_rank; ++r) a = fmaf(qa[r], T::one(cc[s * p.kv_rank + r]), a);
      for (int r = 0; r < p.rot; ++r) a = fmaf(q[p.dim + r], T::one(rc[s * p.rot + r]), a);
      sc = a * p.scale;
    }
    float mx = wave_max(sc);
    __syncthreads();
    if ((t & 63) == 0) red[t >> 6] = mx;
    __syncthreads();
    mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float mn = fmaxf(m, mx);
    const float keep = expf(m - mn), e = expf(sc - mn);
    pr[t] = e;
    l = l * keep + block_sum256(e, red);  // (barriers: pr is complete)
    m = mn;
    const int n = hi - s0 + 1 < 256 ? (int)(hi - s0 + 1) : 256;
    for (int r = t; r < p.kv_rank; r += 256) {
      float a = o[r] * keep;
      for (int j = 0; j < n; ++j) a = fmaf(pr[j], T::one(cc[(s0 + j) * p.kv_rank + r]), a);
      o[r] = a;
    }
    __syncthreads();
  }
  const float inv = l > 0.f ? 1.f / l : 0.f;
  __syncthreads();
  const S* wv = (const S*)p.w_uv + (long)h * p.vdim * p.kv_rank;
  S* out = (S*)p.out + ((long)tok * p.heads + h) * p.vdim;
  for (int v = t >> 6; v < p.vdim; v += 4) {
    float a = 0.f;
    for (int r = t & 63; r < p.kv_rank; r += 64) a = fmaf(T::one(wv[(long)v * p.kv_rank + r]), o[r], a);
    a = wave_sum(a);
    if ((t & 63) == 0) out[v] = T::pack(a * inv);
  }
}

// ---------------------------------------------------------------------------------------
// decode
// ---------------------------------------------------------------------------------------
// q_abs[tok, h, :] = (Wuk_h^T q_h | rotated part | zeros). Grid (heads, column blocks of 64, token groups of 4):
// eight threads cover 64 columns, 32 thread rows share the head's dim rows.
constexpr int kAbsTok = 4;
template <typename T>
__global__ void __launch_bounds__(256) latent_absorb_kernel(const LatentParams p) {
  __shared__ float part[32][64 + 4];
  const int h = blockIdx.x, t = threadIdx.x, cg = t & 7, dg = t >> 3;
  const int tokens = p.batch * p.t, tok0 = blockIdx.z * kAbsTok;
  const int col = blockIdx.y * 64 + cg * 8;
  const int hd = p.dim + p.rot;
  const uint16_t* wk = (const uint16_t*)p.w_uk + (long)h * p.dim * p.kv_rank;
  float acc[kAbsTok][8];
#pragma unroll
  for (int j = 0; j < kAbsTok; ++j)
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[j][i] = 0.f;
  if (col < p.kv_rank) {
#pragma unroll 4
    for (int d = dg; d < p.dim; d += 32) {
      float w[8];
      unpack8<T>(ld16_stream(wk + (long)d * p.kv_rank + col), w);
#pragma unroll
      for (int j = 0; j < kAbsTok; ++j) {
        const int tok = tok0 + j < tokens ? tok0 + j : tokens - 1;
        const float q = T::one(((const uint16_t*)p.q)[((long)tok * p.heads + h) * hd + d]);
#pragma unroll
        for (int i = 0; i < 8; ++i) acc[j][i] = fmaf(w[i], q, acc[j][i]);
      }
    }
  }
#pragma unroll
  for (int j = 0; j < kAbsTok; ++j) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 8; ++i) part[dg][cg * 8 + i] = acc[j][i];
    __syncthreads();
    const int tok = tok0 + j;
    if (tok < tokens && t < 64) {
      float a = 0.f;
#pragma unroll
      for (int d = 0; d < 32; ++d) a += part[d][t];
      const int c = blockIdx.y * 64 + t;
      uint16_t* dst = (uint16_t*)p.q_abs + ((long)tok * p.heads + h) * p.kp;
      if (c < p.kv_rank) dst[c] = T::pack(a);
    }
    if (tok < tokens && blockIdx.y == 0) {  // the part behind the latent columns: rotation, zeros
      const uint16_t* qh = (const uint16_t*)p.q + ((long)tok * p.heads + h) * hd;
      uint16_t* dst = (uint16_t*)p.q_abs + ((long)tok * p.heads + h) * p.kp;
      for (int c = p.kv_rank + t; c < p.kp; c += 256)
        dst[c] = c < p.kv_rank + p.rot
                     ? T::pack(rotated_q<T>(qh, p.cos_sin + (long)tok * p.rot, p.dim, p.rot, p.dim + c - p.kv_rank))
                     : (uint16_t)0;
    }
  }
}

// Splits of token tok that hold visible keys: the grid covers the largest span, the rest leave at once
__device__ __forceinline__ int live_splits(const LatentParams& p, long lo, long hi) {
  return hi < lo ? 0 : (int)((hi - lo) / p.split_keys) + 1;
}

// Grid (splits, groups of 16 HT heads, tokens); eight waves, 64 keys per block; the queries and all of a block's
// rows are requested at once.
//   scores: wave w takes keys 16 (w % 4) .. and head tile w / 4: A = key rows, B = the 16 heads' queries; lane
//           (g, i) ends up with head i, keys 16 (w % 4) + 4 g + r
//   values: O^T[rank, head] += C^T P^T, the latent rows read back transposed; wave w owns the rank
//           tiles w, w + 8, ... of all head tiles; contraction slots of lane group g: keys 4 g + r and
//           16 + 4 g + r of 32
constexpr int kDecKeys = 64, kDecThreads = 512;
constexpr int kMaxDecodeWidth = 576;  // kv_rank + rot, rounded up to 64
template <typename T, int NT, int HT>  // kv_rank <= 128 NT
__global__ void __launch_bounds__(kDecThreads) latent_decode_kernel(const LatentParams p) {
  constexpr int KG = 2 * NT + 1, HEADS = 16 * HT;  // blocks of 64 columns (kv_rank + rot <= 128 NT + 64)
  __shared__ float mred[4][HEADS], lred[4][HEADS];
  __shared__ __align__(16) uint16_t pl[HEADS][kDecKeys + 8];
  uint16_t* cl = (uint16_t*)la_smem;    // [kp / 64][64 keys][64]
  uint16_t* ql = cl + kDecKeys * p.kp;  // [kp / 64][HEADS][64]
  const int t = threadIdx.x, lane = t & 63, wave = __builtin_amdgcn_readfirstlane(t >> 6), g = lane >> 4, i16 = lane & 15;
  const int split = blockIdx.x, h0 = blockIdx.y * HEADS, tok = blockIdx.z, b = tok / p.t;
  long lo, hi;
  visible(p, tok, b, lo, hi);
  if (split >= live_splits(p, lo, hi)) return;  // uniform for the workgroup
  const long s_begin = lo + (long)split * p.split_keys;
  long s_end = s_begin + p.split_keys;  // exclusive
  s_end = s_end < hi + 1 ? s_end : hi + 1;
  const uint16_t* cc = (const uint16_t*)p.c_cache + b * p.c_batch;
  const uint16_t* rc = (const uint16_t*)p.r_cache + b * p.r_batch;
  const bool rot8 = p.rot % 8 == 0;
  const int lrow = lane >> 3;
  {  // the heads' queries: eight rows per instruction, the instructions dealt out to the waves
    constexpr int QB = HEADS / 8;
    const int qb = wave % QB, row = qb * 8 + lrow, hh = h0 + row < p.heads ? h0 + row : p.heads - 1;
    const uint16_t* src = (const uint16_t*)p.q_abs + ((long)tok * p.heads + hh) * p.kp + ((lane & 7) ^ tile_swz(row)) * 8;
    for (int cb = wave / QB; cb * 64 < p.kp; cb += 8 / QB) load_lds16(src + cb * 64, &ql[(cb * HEADS + qb * 8) * 64]);
  }
  const int width = p.kv_rank + (rot8 ? p.rot : 0);  // columns that are loaded
  f32x4 acc[NT][HT];
  float m[HT], l[HT];
#pragma unroll
  for (int h = 0; h < HT; ++h) {
    m[h] = -1e30f;
    l[h] = 0.f;
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[j][h] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const float sc = p.scale * 1.4426950408889634f;
  const int kt = wave & 3, ht = wave >> 2;  // key tile and head tile of this wave's scores
  // operand addresses: only the block of columns and multiples of 16 rows change, by constants
  const int krow = 16 * kt + i16, kswz = tile_swz(krow);
  const uint16_t *ka = cl + krow * 64 + ((g ^ kswz) << 3), *kb = cl + krow * 64 + (((4 + g) ^ kswz) << 3);
  const int qrow = 16 * (ht < HT ? ht : 0) + i16, qswz = tile_swz(qrow);
  const uint16_t *qa = ql + qrow * 64 + ((g ^ qswz) << 3), *qb = ql + qrow * 64 + (((4 + g) ^ qswz) << 3);
  const int vrow = 4 * g + (i16 >> 2);
  const uint16_t* va = cl + ((wave >> 2) * kDecKeys + vrow) * 64 + (((2 * (wave & 3) + ((i16 & 3) >> 1)) ^ tile_swz(vrow)) << 3) + 4 * (i16 & 1);
  for (long s0 = s_begin; s0 < s_end; s0 += kDecKeys) {
    __syncthreads();  // the previous block is done with
    // wave w delivers rows 8 w ..; rows past the split repeat its last one (their scores are masked), columns
    // past the rows' end repeat their start (the queries hold zeros there)
    {
      const int row = wave * 8 + lrow;
      const long s = s0 + row < s_end ? s0 + row : s_end - 1;
      const uint16_t *crow = cc + s * p.kv_rank, *rrow = rc + s * p.rot - p.kv_rank;
      const int lc = ((lane & 7) ^ tile_swz(row)) * 8;
#pragma unroll
      for (int cb = 0; cb < KG; ++cb) {
        if (cb * 64 >= p.kp) break;
        const int c = cb * 64 + lc < width ? cb * 64 + lc : 0;
        load_lds16((c < p.kv_rank ? crow : rrow) + c, &cl[(cb * kDecKeys + wave * 8) * 64]);
      }
    }
    wait_loads<0>();
    if (!rot8) {  // the rotated part element by element
      __syncthreads();
      for (int c = t; c < kDecKeys * p.rot; c += kDecThreads) {
        const int r = c / p.rot, e = c - r * p.rot;
        const long s = s0 + r < s_end ? s0 + r : s_end - 1;
        cl[tile_at<kDecKeys>(r, p.kv_rank + e)] = rc[s * p.rot + e];
      }
    }
    __syncthreads();
    f32x4 s4 = {0.f, 0.f, 0.f, 0.f}, s5 = {0.f, 0.f, 0.f, 0.f};
    if (ht < HT) {
#pragma unroll
      for (int cb = 0; cb < KG; ++cb) {
        if (cb * 64 < p.kp) {
          s4 = mfma16x16x32<T>(*(const u32x4*)(ka + cb * kDecKeys * 64), *(const u32x4*)(qa + cb * HEADS * 64), s4);
          s5 = mfma16x16x32<T>(*(const u32x4*)(kb + cb * kDecKeys * 64), *(const u32x4*)(qb + cb * HEADS * 64), s5);
        }
      }
      float mx = -INFINITY;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        s4[r] = s0 + 16 * kt + 4 * g + r < s_end ? (s4[r] + s5[r]) * sc : -INFINITY;
        mx = fmaxf(mx, s4[r]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16));
      mx = fmaxf(mx, __shfl_xor(mx, 32));
      if (g == 0) mred[kt][16 * ht + i16] = mx;
    }
    __syncthreads();
    float keep[HT];
#pragma unroll
    for (int h = 0; h < HT; ++h) {
      float mn = m[h];
#pragma unroll
      for (int w = 0; w < 4; ++w) mn = fmaxf(mn, mred[w][16 * h + i16]);
      keep[h] = exp2f(m[h] - mn);
      m[h] = mn;
    }
    if (ht < HT) {
      const float mn = HT == 2 && ht ? m[HT - 1] : m[0];
      float e[4], sum = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) { e[r] = exp2f(s4[r] - mn); sum += e[r]; }
      *(u32x2*)&pl[16 * ht + i16][16 * kt + 4 * g] = u32x2{T::pack2(e[0], e[1]), T::pack2(e[2], e[3])};
      sum += __shfl_xor(sum, 16);
      sum += __shfl_xor(sum, 32);
      if (g == 0) lred[kt][16 * ht + i16] = sum;
    }
    __syncthreads();
#pragma unroll
    for (int h = 0; h < HT; ++h) {
      l[h] = l[h] * keep[h] + ((lred[0][16 * h + i16] + lred[1][16 * h + i16]) + (lred[2][16 * h + i16] + lred[3][16 * h + i16]));
#pragma unroll
      for (int j = 0; j < NT; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[j][h][r] *= keep[h];
    }
#pragma unroll
    for (int kk = 0; kk < kDecKeys / 32; ++kk) {
      u32x4 pb[HT];
#pragma unroll
      for (int h = 0; h < HT; ++h) {
        const u32x2 plo = *(const u32x2*)&pl[16 * h + i16][32 * kk + 4 * g], phi = *(const u32x2*)&pl[16 * h + i16][32 * kk + 16 + 4 * g];
        pb[h] = u32x4{plo.x, plo.y, phi.x, phi.y};
      }
#pragma unroll
      for (int j = 0; j < NT; ++j) {
        if (16 * (wave + 8 * j) < p.kv_rank) {  // uniform; a last tile may reach into the rotated part: never stored
          const u32x2 a0 = lds_read_tr16(va + (2 * j * kDecKeys + 32 * kk) * 64);
          const u32x2 a1 = lds_read_tr16(va + (2 * j * kDecKeys + 32 * kk + 16) * 64);
          const u32x4 a = {a0.x, a0.y, a1.x, a1.y};
#pragma unroll
          for (int h = 0; h < HT; ++h) acc[j][h] = mfma16x16x32<T>(a, pb[h], acc[j][h]);
        }
      }
    }
  }
#pragma unroll
  for (int h = 0; h < HT; ++h) {
    const int hh = h0 + 16 * h + i16;
    if (hh >= p.heads) continue;
    const long at = ((long)tok * p.heads + hh) * p.splits + split;
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      const int c = 16 * (wave + 8 * j) + 4 * g;  // (kv_rank is a multiple of 8)
      if (c < p.kv_rank) *(f32x4*)&p.part[at * p.kv_rank + c] = acc[j][h];
    }
    if (wave == 0 && g == 0) {
      p.part_ml[at * 2] = m[h];
      p.part_ml[at * 2 + 1] = l[h];
    }
  }
}

// Grid (heads, blocks of 32 value rows, tokens): merges the splits of a head, then Wuv_h times the result;
// eight lanes per value row
constexpr int kMaxSplits = 64;
template <typename T>
__global__ void __launch_bounds__(256) latent_output_kernel(const LatentParams p) {
  __shared__ float ws[kMaxSplits];
  float* o = (float*)la_smem;  // kv_rank
  const int h = blockIdx.x, tok = blockIdx.z, t = threadIdx.x;
  const long at = ((long)tok * p.heads + h) * p.splits;
  const float* part = p.part + at * p.kv_rank;
  long lo, hi;
  visible(p, tok, tok / p.t, lo, hi);
  const int live = live_splits(p, lo, hi);
  if (t < kWave) {  // the splits' shares, one per lane
    const bool in = t < live;
    const float mm = in ? p.part_ml[(at + t) * 2] : -1e30f, ll = in ? p.part_ml[(at + t) * 2 + 1] : 0.f;
    const float e = exp2f(mm - wave_max(mm));
    ws[t] = in ? e / wave_sum(e * ll) : 0.f;
  }
  __syncthreads();
  // splits past the live ones repeat the last one with a share of zero: sixteen loads in flight
  for (int r = t; r < p.kv_rank; r += 256) {
    float a = 0.f;
    for (int s0 = 0; s0 < live; s0 += 16) {
      float v[16];
#pragma unroll
      for (int u = 0; u < 16; ++u) v[u] = part[(long)(s0 + u < live ? s0 + u : live - 1) * p.kv_rank + r];
#pragma unroll
      for (int u = 0; u < 16; ++u) a = fmaf(ws[s0 + u], v[u], a);
    }
    o[r] = a;
  }
  __syncthreads();
  const int v = blockIdx.y * 32 + (t >> 3);
  const int vc = v < p.vdim ? v : p.vdim - 1;
  const uint16_t* w = (const uint16_t*)p.w_uv + ((long)h * p.vdim + vc) * p.kv_rank;
  float a = 0.f;
#pragma unroll 8
  for (int c = (t & 7) * 8; c < p.kv_rank; c += 64) {
    float f[8];
    unpack8<T>(ld16_stream(w + c), f);
#pragma unroll
    for (int i = 0; i < 8; ++i) a = fmaf(f[i], o[c + i], a);
  }
  a += dpp_f32<kDppXor1>(a);
  a += dpp_f32<kDppXor2>(a);
  a += dpp_f32<kDppHalfMirror>(a);
  if ((t & 7) == 0 && v < p.vdim) ((uint16_t*)p.out)[((long)tok * p.heads + h) * p.vdim + v] = T::pack(a);
}

// ---------------------------------------------------------------------------------------
// prefill: grid (heads, tiles of 32 NW queries, longest first) of one batch row; NW waves of 32 queries, two or more
// workgroups per CU. LDS holds two stages of 64 keys and one of their values: while block s is multiplied with
// the queries, its values and the keys of block s + 1 are on their way (LDS-direct loads, no registers).
// ---------------------------------------------------------------------------------------
template <int DKC, int DVT, int NW>
constexpr size_t latent_prefill_lds() {  // K stage, then (the queries, before the loop | second K stage, V)
  constexpr size_t k = (size_t)64 * DKC * 32 * 2, v = (size_t)64 * DVT * 16 * 2, q = (size_t)32 * NW * DKC * 32 * 2;
  return k + (q > k + v ? q : k + v);
}
template <typename T, int DKC, int DVT, int NW>
__global__ void __launch_bounds__(64 * NW, DKC > 6 ? 1 : 2) latent_prefill_kernel(const LatentParams p) {
  static_assert(DKC % 2 == 0 && DVT % 4 == 0 && (NW == 2 || NW == 4), "tiles of 64 columns");
  constexpr int QT = 32 * NW, KG = DKC / 2, VG = DVT / 4;  // queries per workgroup, blocks of 64 columns
  constexpr int RB = 8 / NW, RSTEP = 8 * NW;               // blocks of eight rows per wave, rows between them
  constexpr int KSTAGE = KG * 64 * 64;
  uint16_t* smem = (uint16_t*)la_smem;
  uint16_t* vl = smem + 2 * KSTAGE;
  uint16_t* ql = smem + KSTAGE;  // [KG][QT][64], until the loop starts
  const int t = threadIdx.x, lane = t & 63, wave = __builtin_amdgcn_readfirstlane(t >> 6), g = lane >> 4, i16 = lane & 15;
  const int h = blockIdx.x, qt0 = ((int)gridDim.y - 1 - (int)blockIdx.y) * QT;
  const int hd = p.dim + p.rot, dk = hd;
  const long first_row = p.row_start ? p.row_start[p.b0] : 0;
  f32x4 acc[2][DVT];
  float m[2] = {-1e30f, -1e30f}, l[2] = {0.f, 0.f};
#pragma unroll
  for (int qt = 0; qt < 2; ++qt)
#pragma unroll
    for (int j = 0; j < DVT; ++j) acc[qt][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const float sc = p.scale * 1.4426950408889634f;
  const int q_last = (qt0 + QT < p.t ? qt0 + QT : p.t) - 1;
  const long hi = (long)p.q_first + q_last;
  long lo = p.window > 0 ? (long)p.q_first + qt0 - p.window + 1 : 0;
  lo = lo > first_row ? lo : first_row;
  lo = lo > p.kv_first ? lo : p.kv_first;
  const int kvp = p.heads * (p.dim + p.vdim);
  // key / value rows counted from lo
  const uint16_t* kbase = (const uint16_t*)p.kv + (lo - p.kv_first) * kvp + (long)h * p.dim;
  const uint16_t* vbase = (const uint16_t*)p.kv + (lo - p.kv_first) * kvp + (long)p.heads * p.dim + (long)h * p.vdim;
  const uint16_t* rc = (const uint16_t*)p.r_cache + p.b0 * p.r_batch + lo * p.rot;
  const int n_keys = hi >= lo ? (int)(hi - lo + 1) : 0;
  const bool vec = p.dim % 8 == 0 && p.rot % 8 == 0 && p.vdim % 8 == 0;  // 16-byte chunks stay aligned
  // Wave w delivers rows 8 w .., 8 (w + NW) .., ... of a block (their swizzles agree). Rows past the last key
  // repeat it (masked), columns past a key's end repeat its start (the queries hold zeros there), columns
  // past a value's end are never stored.
  const int lrow = wave * 8 + (lane >> 3), lc = ((lane & 7) ^ tile_swz(lrow)) * 8;
  auto load_k = [&](int s0, uint16_t* dst) {
    if (vec) {
#pragma unroll
      for (int u = 0; u < RB; ++u) {
        const long row = s0 + lrow + RSTEP * u < n_keys ? s0 + lrow + RSTEP * u : n_keys - 1;
#pragma unroll
        for (int cg = 0; cg < KG; ++cg) {
          const int c = cg * 64 + lc < dk ? cg * 64 + lc : 0;
          load_lds16(c < p.dim ? kbase + row * kvp + c : rc + row * p.rot + (c - p.dim),
                     &dst[(cg * 64 + wave * 8 + RSTEP * u) * 64]);
        }
      }
    } else {
      for (int c = t; c < 64 * DKC * 32; c += 64 * NW) {
        const int r = c / (DKC * 32), e = c - r * DKC * 32;
        const long row = s0 + r < n_keys ? s0 + r : n_keys - 1;
        dst[tile_at<64>(r, e)] = e < p.dim ? kbase[row * kvp + e] : (e < dk ? rc[row * p.rot + e - p.dim] : (uint16_t)0);
      }
    }
  };
  auto load_v = [&](int s0) {
    if (vec) {
#pragma unroll
      for (int u = 0; u < RB; ++u) {
        const long row = s0 + lrow + RSTEP * u < n_keys ? s0 + lrow + RSTEP * u : n_keys - 1;
#pragma unroll
        for (int cg = 0; cg < VG; ++cg)
          load_lds16(vbase + row * kvp + (cg * 64 + lc < p.vdim ? cg * 64 + lc : 0), &vl[(cg * 64 + wave * 8 + RSTEP * u) * 64]);
      }
    } else {
      for (int c = t; c < 64 * DVT * 16; c += 64 * NW) {
        const int r = c / (DVT * 16), e = c - r * DVT * 16;
        const long row = s0 + r < n_keys ? s0 + r : n_keys - 1;
        vl[tile_at<64>(r, e)] = e < p.vdim ? vbase[row * kvp + e] : (uint16_t)0;
      }
    }
  };
  if (n_keys > 0) load_k(0, smem);
  // queries: rotated, rounded, through LDS into operand registers (column i16, k-chunk g)
  const bool qvec = p.dim % 8 == 0 && p.rot % 16 == 0;
#pragma unroll 4
  for (int c = t; c < QT * DKC * 4; c += 64 * NW) {
    const int r = c / (DKC * 4), e0 = (c - r * DKC * 4) * 8;
    const long tok = (long)p.b0 * p.t + (qt0 + r < p.t ? qt0 + r : p.t - 1);
    *(u32x4*)&ql[tile_at<QT>(r, e0)] =
        rotated_q8<T>((const uint16_t*)p.q + (tok * p.heads + h) * hd, p.cos_sin + tok * p.rot, p.dim, p.rot, e0, qvec);
  }
  __syncthreads();
  u32x4 q[2][DKC];
#pragma unroll
  for (int qt = 0; qt < 2; ++qt)
#pragma unroll
    for (int c = 0; c < DKC; ++c) q[qt][c] = *(const u32x4*)&ql[tile_at<QT>(wave * 32 + qt * 16 + i16, c * 32 + 8 * g)];
  // this wave's queries, as positions counted from lo
  const int wq0 = (int)((long)p.q_first + qt0 + wave * 32 - lo), wq1 = wq0 + 31;
  for (int s0 = 0, buf = 0; s0 < n_keys; s0 += 64, buf ^= 1) {
    const uint16_t* kl = smem + buf * KSTAGE;
    const bool more = s0 + 64 < n_keys;
    // (blocks that none of the wave's queries sees are skipped)
    const bool mine = s0 <= wq1 && (p.window <= 0 || s0 + 63 > wq0 - p.window);
    wait_loads<0>();  // this wave's rows of the keys have landed
    __syncthreads();                     // ... and everybody's; everybody is done with the values and the other keys
    load_v(s0);
    if (more) load_k(s0 + 64, smem + (buf ^ 1) * KSTAGE);
    u32x4 pb[2][2];
    if (mine) {
      f32x4 s4[2][4];
#pragma unroll
      for (int kt = 0; kt < 4; ++kt) {
#pragma unroll
        for (int qt = 0; qt < 2; ++qt) s4[qt][kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int c = 0; c < DKC; ++c) {
          const u32x4 a = *(const u32x4*)&kl[tile_at<64>(kt * 16 + i16, c * 32 + 8 * g)];
#pragma unroll
          for (int qt = 0; qt < 2; ++qt) s4[qt][kt] = mfma16x16x32<T>(a, q[qt][c], s4[qt][kt]);
        }
      }
      const bool full = s0 + 63 <= wq0 && (p.window <= 0 || s0 >= wq1 - p.window + 1);
#pragma unroll
      for (int qt = 0; qt < 2; ++qt) {
        float mx = -INFINITY;
        if (full) {
#pragma unroll
          for (int kt = 0; kt < 4; ++kt)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              s4[qt][kt][r] *= sc;
              mx = fmaxf(mx, s4[qt][kt][r]);
            }
        } else {
          // keys counted from the block's start: the last one seen, and the last one in front of the window
          const int last = wq0 + qt * 16 + i16 - s0, before = p.window > 0 ? last - p.window : -1;
#pragma unroll
          for (int kt = 0; kt < 4; ++kt)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              const int s = kt * 16 + 4 * g + r;
              const float v = s4[qt][kt][r] * sc;
              s4[qt][kt][r] = s <= last && s > before ? v : -INFINITY;
              mx = fmaxf(mx, s4[qt][kt][r]);
            }
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16));
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        if (__any(mx > m[qt])) {
          const float mn = fmaxf(m[qt], mx), keep = __builtin_amdgcn_exp2f(m[qt] - mn);
          m[qt] = mn;
          l[qt] *= keep;
#pragma unroll
          for (int j = 0; j < DVT; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) acc[qt][j][r] *= keep;
        }
        float e[4][4], sum = 0.f;
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            e[kt][r] = __builtin_amdgcn_exp2f(s4[qt][kt][r] - m[qt]);
            sum += e[kt][r];
          }
        l[qt] += sum;  // this lane's keys only; the lane groups are added up at the end
#pragma unroll
        for (int kk = 0; kk < 2; ++kk)
          pb[qt][kk] = u32x4{T::pack2(e[2 * kk][0], e[2 * kk][1]), T::pack2(e[2 * kk][2], e[2 * kk][3]),
                             T::pack2(e[2 * kk + 1][0], e[2 * kk + 1][1]), T::pack2(e[2 * kk + 1][2], e[2 * kk + 1][3])};
      }
    }
    // the values were requested before the next keys
    if (more) wait_loads<RB * KG>();
    else wait_loads<0>();
    __syncthreads();
    if (mine) {
#pragma unroll
      for (int kk = 0; kk < 2; ++kk)
#pragma unroll
        for (int j = 0; j < DVT; ++j) {
          const int row = 32 * kk + 4 * g + (i16 >> 2), col = 16 * j + 4 * (i16 & 3);
          const u32x2 a0 = lds_read_tr16(&vl[tile_at<64>(row, col)]);
          const u32x2 a1 = lds_read_tr16(&vl[tile_at<64>(row + 16, col)]);
          const u32x4 va = {a0.x, a0.y, a1.x, a1.y};
#pragma unroll
          for (int qt = 0; qt < 2; ++qt) acc[qt][j] = mfma16x16x32<T>(va, pb[qt][kk], acc[qt][j]);
        }
    }
  }
#pragma unroll
  for (int qt = 0; qt < 2; ++qt) {
    float s = l[qt];
    s += __shfl_xor(s, 16);
    s += __shfl_xor(s, 32);
    const float inv = s > 0.f ? 1.f / s : 0.f;
    const int tq = qt0 + wave * 32 + qt * 16 + i16;
    if (tq >= p.t) continue;
    uint16_t* dst = (uint16_t*)p.out + (((long)p.b0 * p.t + tq) * p.heads + h) * p.vdim;
#pragma unroll
    for (int j = 0; j < DVT; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int v = 16 * j + 4 * g + r;
        if (v < p.vdim) dst[v] = T::pack(acc[qt][j][r] * inv);
      }
  }
}

// ---------------------------------------------------------------------------------------
// launchers
// ---------------------------------------------------------------------------------------
template <typename T>
static int launch_latent_plain(hipStream_t s, const LatentParams& p) {
  const size_t lds = ((size_t)p.dim + p.rot + 2 * (size_t)p.kv_rank + 256) * 4;
  if (p.batch * p.t > 65535) return MUI_ERR_UNSUPPORTED;
  return launch_with_lds(latent_plain_kernel<T>, dim3(p.heads, p.batch * p.t), dim3(256), lds, s, p);
}

template <typename T, int HT>
static int launch_latent_decode_h(hipStream_t s, const LatentParams& p) {
  const dim3 grid(p.splits, ceil_div(p.heads, 16 * HT), p.batch * p.t), block(kDecThreads);
  const size_t lds = (size_t)(kDecKeys + 16 * HT) * p.kp * 2;
  if (p.kp <= 192 && p.kv_rank <= 128) return launch_with_lds(latent_decode_kernel<T, 1, HT>, grid, block, lds, s, p);
  if (p.kp <= 320 && p.kv_rank <= 256) return launch_with_lds(latent_decode_kernel<T, 2, HT>, grid, block, lds, s, p);
  return launch_with_lds(latent_decode_kernel<T, 4, HT>, grid, block, lds, s, p);
}

template <typename T>
static int launch_latent_decode(hipStream_t s, const LatentParams& p) {
  const int tokens = p.batch * p.t;
  if (tokens > 65535 || p.kp > kMaxDecodeWidth) return MUI_ERR_UNSUPPORTED;
  hipLaunchKernelGGL((latent_absorb_kernel<T>), dim3(p.heads, ceil_div(p.kv_rank, 64), ceil_div(tokens, kAbsTok)),
                     dim3(256), 0, s, p);
  const int st = p.heads > 16 ? launch_latent_decode_h<T, 2>(s, p) : launch_latent_decode_h<T, 1>(s, p);
  if (st != MUI_OK) return st;
  return launch_with_lds(latent_output_kernel<T>, dim3(p.heads, ceil_div(p.vdim, 32), tokens), dim3(256),
                         (size_t)p.kv_rank * 4, s, p);
}

template <typename T, int DKC, int DVT, int NW>
static int launch_latent_prefill_w(hipStream_t s, const LatentParams& p) {
  const int tiles = ceil_div(p.t, 32 * NW);
  if (tiles > 65535) return MUI_ERR_UNSUPPORTED;
  return launch_with_lds(latent_prefill_kernel<T, DKC, DVT, NW>, dim3(p.heads, tiles), dim3(64 * NW),
                         latent_prefill_lds<DKC, DVT, NW>(), s, p);
}

template <typename T, int DKC, int DVT>
static int launch_latent_prefill_t(hipStream_t s, const LatentParams& p) {
  // short prompts: half as many queries per workgroup, so that there are workgroups for every CU
  if (p.heads * ceil_div(p.t, 128) <= device_cus()) return launch_latent_prefill_w<T, DKC, DVT, 2>(s, p);
  return launch_latent_prefill_w<T, DKC, DVT, 4>(s, p);
}

static bool prefill_covers(int dk, int vdim) { return dk <= 256 && vdim <= 256; }

template <typename T>
static int launch_latent_prefill(hipStream_t s, const LatentParams& p) {
  const int dk = p.dim + p.rot;
  if (dk <= 64 && p.vdim <= 64) return launch_latent_prefill_t<T, 2, 4>(s, p);
  if (dk <= 128 && p.vdim <= 128) return launch_latent_prefill_t<T, 4, 8>(s, p);
  if (dk <= 192 && p.vdim <= 128) return launch_latent_prefill_t<T, 6, 8>(s, p);
  if (prefill_covers(dk, p.vdim)) return launch_latent_prefill_t<T, 8, 16>(s, p);
  return MUI_ERR_UNSUPPORTED;
}

}  // namespace mui

using namespace mui;

extern "C" int mui_latent_prepare(mui_stream_t stream, int dtype, const void* down, long down_pitch, const void* q_gain,
                                  const void* kv_gain, float epsilon, const double* inv_freq,
                                  const int64_t* cache_position, const int64_t* row_start, void* q_latent,
                                  float* cos_sin, void* c_cache, long c_batch_stride, void* r_cache,
                                  long r_batch_stride, int batch, int t, int q_rank, int kv_rank, int rot_dim,
                                  int max_cache_len) {
  MUI_CHECK_ARG(down && q_gain && cache_position && q_latent && cos_sin && batch > 0 && t > 0 && q_rank > 0);
  MUI_CHECK_ARG(kv_rank > 0 && rot_dim >= 0 && rot_dim % 2 == 0 && (rot_dim == 0 || inv_freq));
  MUI_CHECK_ARG(!kv_gain || (c_cache && r_cache && max_cache_len > 0));
  MUI_CHECK_ARG(down_pitch >= q_rank + (kv_gain ? kv_rank + rot_dim : 0));
  LatentParams p = {};
  p.down = down; p.down_pitch = down_pitch; p.q_gain = q_gain; p.kv_gain = kv_gain; p.eps = epsilon;
  p.inv_freq = inv_freq; p.cache_position = cache_position; p.row_start = row_start; p.q_latent = q_latent;
  p.cos_sin = cos_sin; p.c_cache = c_cache; p.c_batch = c_batch_stride; p.r_cache = r_cache; p.r_batch = r_batch_stride;
  p.batch = batch; p.t = t; p.q_rank = q_rank; p.kv_rank = kv_rank; p.rot = rot_dim; p.max_cache_len = max_cache_len;
  hipStream_t s = (hipStream_t)stream;
  const dim3 grid(batch * t), block(256);
  if (dtype == MUI_DTYPE_F16) hipLaunchKernelGGL((latent_prepare_kernel<F16>), grid, block, 0, s, p);
  else if (dtype == MUI_DTYPE_BF16) hipLaunchKernelGGL((latent_prepare_kernel<BF16>), grid, block, 0, s, p);
  else if (dtype == MUI_DTYPE_F32) hipLaunchKernelGGL((latent_prepare_kernel<F32>), grid, block, 0, s, p);
  else return MUI_ERR_INVALID_ARG;
  return launch_status();
}

static int latent_kp(int kv_rank, int rot_dim) { return (kv_rank + rot_dim + 63) / 64 * 64; }

// keys per split and number of splits of the decode kernel for spans of up to `span` keys
static void latent_split(int batch, int t, int heads, int span, int* splits, int* split_keys) {
  const int groups = batch * t * ceil_div(heads, heads > 16 ? 32 : 16);
  int want = device_cus() * 2 / (groups > 0 ? groups : 1);
  want = want < 1 ? 1 : (want > kMaxSplits ? kMaxSplits : want);
  const int blocks = ceil_div(span, kDecKeys);
  const int per = ceil_div(blocks, want);
  *split_keys = per * kDecKeys;
  *splits = ceil_div(blocks, per);
}

extern "C" int mui_latent_attention_route(int dtype, int tokens, int heads, int dim, int rot_dim, int vdim, int kv_rank) {
  if (dtype == MUI_DTYPE_F32 || kv_rank % 8) return MUI_LATENT_PLAIN;
  if (tokens > MUI_MAX_TOKENS && prefill_covers(dim + rot_dim, vdim)) return MUI_LATENT_PREFILL;
  return latent_kp(kv_rank, rot_dim) <= kMaxDecodeWidth ? MUI_LATENT_DECODE : MUI_LATENT_PLAIN;
}

extern "C" size_t mui_latent_decode_scratch_bytes(int batch, int t, int heads, int kv_rank, int rot_dim, int span) {
  if (batch < 1 || t < 1 || heads < 1 || span < 1) return 0;
  int splits, keys;
  latent_split(batch, t, heads, span, &splits, &keys);
  const size_t q = ((size_t)batch * t * heads * latent_kp(kv_rank, rot_dim) * 2 + 255) / 256 * 256;
  return q + (size_t)batch * t * heads * splits * (kv_rank + 2) * 4;
}

extern "C" int mui_latent_attention(mui_stream_t stream, int dtype, int route, const void* q, const float* cos_sin,
                                    const void* w_uk, const void* w_uv, const void* c_cache, long c_batch_stride,
                                    const void* r_cache, long r_batch_stride, const int64_t* cache_position,
                                    const int64_t* row_start, float scale, int window, void* scratch, int span,
                                    void* out, int batch, int t, int heads, int dim, int rot_dim, int vdim, int kv_rank,
                                    int max_cache_len) {
  MUI_CHECK_ARG(q && cos_sin && w_uk && w_uv && c_cache && r_cache && cache_position && out);
  MUI_CHECK_ARG(batch > 0 && t > 0 && heads > 0 && dim > 0 && rot_dim >= 0 && vdim > 0 && kv_rank > 0 && max_cache_len > 0);
  LatentParams p = {};
  p.q = q; p.cos_sin = (float*)cos_sin; p.w_uk = w_uk; p.w_uv = w_uv; p.c_cache = (void*)c_cache; p.c_batch = c_batch_stride;
  p.r_cache = (void*)r_cache; p.r_batch = r_batch_stride; p.cache_position = cache_position; p.row_start = row_start;
  p.scale = scale; p.window = window; p.out = out; p.batch = batch; p.t = t; p.heads = heads; p.dim = dim; p.rot = rot_dim;
  p.vdim = vdim; p.kv_rank = kv_rank; p.max_cache_len = max_cache_len;
  hipStream_t s = (hipStream_t)stream;
  if (route == MUI_LATENT_PLAIN) {
    if (dtype == MUI_DTYPE_F16) return launch_latent_plain<F16>(s, p);
    if (dtype == MUI_DTYPE_BF16) return launch_latent_plain<BF16>(s, p);
    if (dtype == MUI_DTYPE_F32) return launch_latent_plain<F32>(s, p);
    return MUI_ERR_INVALID_ARG;
  }
  MUI_CHECK_ARG(route == MUI_LATENT_DECODE && scratch && span > 0);
  if (kv_rank % 8 || latent_kp(kv_rank, rot_dim) > kMaxDecodeWidth) return MUI_ERR_UNSUPPORTED;
  if (!aligned16(w_uk) || !aligned16(w_uv) || !aligned16(c_cache) || !aligned16(r_cache) || c_batch_stride % 8 ||
      (rot_dim % 8 == 0 && r_batch_stride % 8) || ((uintptr_t)scratch & 255))
    return MUI_ERR_ALIGNMENT;
  p.kp = latent_kp(kv_rank, rot_dim);
  latent_split(batch, t, heads, span, &p.splits, &p.split_keys);
  p.q_abs = scratch;
  p.part = (float*)((char*)scratch + ((size_t)batch * t * heads * p.kp * 2 + 255) / 256 * 256);
  p.part_ml = p.part + (size_t)batch * t * heads * p.splits * kv_rank;
  if (dtype == MUI_DTYPE_F16) return launch_latent_decode<F16>(s, p);
  if (dtype == MUI_DTYPE_BF16) return launch_latent_decode<BF16>(s, p);
  return MUI_ERR_INVALID_ARG;
}

extern "C" int mui_latent_prefill_attention(mui_stream_t stream, int dtype, const void* q, const float* cos_sin,
                                            const void* kv, int kv_first, int kv_rows, const void* r_cache,
                                            long r_batch_stride, const int64_t* row_start, float scale, int window,
                                            int q_first, void* out, int batch_row, int t, int heads, int dim, int rot_dim,
                                            int vdim) {
  MUI_CHECK_ARG(q && cos_sin && kv && r_cache && out && batch_row >= 0 && t > 0 && heads > 0 && dim > 0 && rot_dim >= 0);
  MUI_CHECK_ARG(vdim > 0 && kv_first >= 0 && kv_rows > 0 && q_first >= kv_first && q_first + t == kv_first + kv_rows);
  MUI_CHECK_ARG(kv_first == 0 || (window > 0 && q_first - window + 1 >= kv_first));
  if (!aligned16(kv) || !aligned16(r_cache) || (rot_dim % 8 == 0 && r_batch_stride % 8)) return MUI_ERR_ALIGNMENT;
  LatentParams p = {};
  p.q = q; p.cos_sin = (float*)cos_sin; p.kv = kv; p.kv_first = kv_first; p.kv_rows = kv_rows; p.r_cache = (void*)r_cache;
  p.r_batch = r_batch_stride; p.row_start = row_start; p.scale = scale; p.window = window; p.q_first = q_first; p.out = out;
  p.b0 = batch_row; p.t = t; p.heads = heads; p.dim = dim; p.rot = rot_dim; p.vdim = vdim;
  if (dtype == MUI_DTYPE_F16) return launch_latent_prefill<F16>((hipStream_t)stream, p);
  if (dtype == MUI_DTYPE_BF16) return launch_latent_prefill<BF16>((hipStream_t)stream, p);
  return MUI_ERR_INVALID_ARG;
}
