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
// formed in double precision (position * inv_freq, reduced modulo 2 pi) and rounded to fp32 once.
#include "skinny.cuh"

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
  float* part;       // decode: [tokens, heads, splits, kv_rank + 2]
  int kp, splits, split_keys;

  const void* kv;    // prefill: [keys, heads * (dim + vdim)], key row 0 = slot kv_first
  int kv_first, kv_rows, q_first, b0;
};

__device__ __forceinline__ void rope_angle(double pos, double inv_freq, float& c, float& s) {
  const double two_pi = 6.283185307179586476925286766559;
  double a = pos * inv_freq;
  a -= two_pi * rint(a / two_pi);
  sincosf((float)a, &s, &c);
}

__device__ __forceinline__ float block_sum256(float v, float* red) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & (kWave - 1)) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return (red[0] + red[1]) + (red[2] + red[3]);
}

// ---------------------------------------------------------------------------------------
// prepare: one workgroup per token
// ---------------------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256) latent_prepare_kernel(const LatentParams p) {
  typedef typename T::storage S;
  __shared__ float red[4];
  const int tok = blockIdx.x, b = tok / p.t, t = threadIdx.x;
  const S* row = (const S*)p.down + (long)tok * p.down_pitch;
  const long slot = p.cache_position[tok - b * p.t];
  const long pos = slot - (p.row_start ? p.row_start[b] : 0);
  float ss = 0.f;
  for (int i = t; i < p.q_rank; i += 256) {
    const float v = T::one(row[i]);
    ss = fmaf(v, v, ss);
  }
  float rs = rsqrtf(block_sum256(ss, red) / (float)p.q_rank + p.eps);
  S* ql = (S*)p.q_latent + (long)tok * p.q_rank;
  for (int i = t; i < p.q_rank; i += 256) ql[i] = T::pack(T::one(((const S*)p.q_gain)[i]) * (T::one(row[i]) * rs));
  const bool kv = p.kv_gain != nullptr && slot >= 0 && slot < p.max_cache_len;
  const int half = p.rot >> 1;
  const S* kr = row + p.q_rank + p.kv_rank;
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
  if (!kv) return;  // uniform for the workgroup
  const S* cr = row + p.q_rank;
  ss = 0.f;
  for (int i = t; i < p.kv_rank; i += 256) {
    const float v = T::one(cr[i]);
    ss = fmaf(v, v, ss);
  }
  rs = rsqrtf(block_sum256(ss, red) / (float)p.kv_rank + p.eps);
  S* dst = (S*)p.c_cache + b * p.c_batch + slot * p.kv_rank;
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

// Grid (splits, head groups of 16, tokens); four waves. 64 keys per block in LDS, rows of kp + 8 elements.
//   scores: wave w takes keys 16 w ..: A = key rows, B = the 16 heads' queries; lane (g, i) ends up with
//           head i, keys 16 w + 4 g + r
//   values: O^T[rank, head] += C^T P^T, the latent rows read back transposed; wave w owns the rank
//           tiles w, w + 4, ...; contraction slots of lane group g: keys 4 g + r and 16 + 4 g + r of 32
template <typename T, int NT>
__global__ void __launch_bounds__(256) latent_decode_kernel(const LatentParams p) {
  __shared__ float mred[4][16], lred[4][16];
  __shared__ __align__(16) uint16_t pl[16][64 + 8];
  const int pitch = p.kp + 8;
  uint16_t* cl = (uint16_t*)la_smem;  // [64][pitch]
  uint16_t* ql = cl + 64 * pitch;     // [16][pitch]
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, g = lane >> 4, i16 = lane & 15;
  const int split = blockIdx.x, h0 = blockIdx.y * 16, tok = blockIdx.z, b = tok / p.t;
  long lo, hi;
  visible(p, tok, b, lo, hi);
  const long s_begin = lo + (long)split * p.split_keys;
  long s_end = s_begin + p.split_keys;  // exclusive
  s_end = s_end < hi + 1 ? s_end : hi + 1;
  const int cpr = p.kp >> 3;
  const u32x4 zero = {0u, 0u, 0u, 0u};
  {
    const int r = t >> 4;  // 16 threads per head
    const int hh = h0 + r < p.heads ? h0 + r : p.heads - 1;
    const uint16_t* src = (const uint16_t*)p.q_abs + ((long)tok * p.heads + hh) * p.kp;
#pragma unroll 5
    for (int c = t & 15; c < cpr; c += 16) *(u32x4*)&ql[r * pitch + c * 8] = ld16(src + c * 8);
  }
  const uint16_t* cc = (const uint16_t*)p.c_cache + b * p.c_batch;
  const uint16_t* rc = (const uint16_t*)p.r_cache + b * p.r_batch;
  const bool rot8 = p.rot % 8 == 0;
  f32x4 acc[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -1e30f, l = 0.f;
  const float sc = p.scale * 1.4426950408889634f;
  for (long s0 = s_begin; s0 < s_end; s0 += 64) {
    __syncthreads();  // the previous block is done with
    // eight threads per key, keys t / 8 and t / 8 + 32; up to ten loads requested together
    const int kr = t >> 3;
    long key[2];
    bool live[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      key[u] = s0 + kr + 32 * u;
      live[u] = key[u] < s_end;
      key[u] = live[u] ? key[u] : s_end - 1;
    }
    for (int c0 = t & 7; c0 < cpr; c0 += 8 * 5) {
      u32x4 v[5][2];
#pragma unroll
      for (int j = 0; j < 5; ++j) {
        const int k = (c0 + 8 * j) * 8;
        const bool in_c = k + 8 <= p.kv_rank, in_r = rot8 && !in_c && k < p.kv_rank + p.rot;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          const uint16_t* src = in_r ? rc + key[u] * p.rot + (k - p.kv_rank) : cc + key[u] * p.kv_rank + (in_c ? k : 0);
          v[j][u] = ld16(src);
          v[j][u] = live[u] && (in_c || in_r) ? v[j][u] : zero;
        }
      }
#pragma unroll
      for (int j = 0; j < 5; ++j)
        if (c0 + 8 * j < cpr)
#pragma unroll
          for (int u = 0; u < 2; ++u) *(u32x4*)&cl[(kr + 32 * u) * pitch + (c0 + 8 * j) * 8] = v[j][u];
    }
    if (!rot8) {
      __syncthreads();
      for (int c = t; c < 64 * p.rot; c += 256) {
        const int r = c / p.rot, e = c - r * p.rot;
        if (s0 + r < s_end) cl[r * pitch + p.kv_rank + e] = rc[(s0 + r) * p.rot + e];
      }
    }
    __syncthreads();
    f32x4 s4 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 6
    for (int k = 0; k < p.kp; k += 32) {
      const u32x4 a = *(const u32x4*)&cl[(16 * wave + i16) * pitch + k + 8 * g];
      const u32x4 q = *(const u32x4*)&ql[i16 * pitch + k + 8 * g];
      s4 = mfma16x16x32<T>(a, q, s4);
    }
    float mx = -INFINITY;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      s4[r] = s0 + 16 * wave + 4 * g + r < s_end ? s4[r] * sc : -INFINITY;
      mx = fmaxf(mx, s4[r]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16));
    mx = fmaxf(mx, __shfl_xor(mx, 32));
    if (g == 0) mred[wave][i16] = mx;
    __syncthreads();
    const float mn = fmaxf(m, fmaxf(fmaxf(mred[0][i16], mred[1][i16]), fmaxf(mred[2][i16], mred[3][i16])));
    const float keep = exp2f(m - mn);
    m = mn;
    float e[4], sum = 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) { e[r] = exp2f(s4[r] - mn); sum += e[r]; }
    *(u32x2*)&pl[i16][16 * wave + 4 * g] = u32x2{T::pack2(e[0], e[1]), T::pack2(e[2], e[3])};
    sum += __shfl_xor(sum, 16);
    sum += __shfl_xor(sum, 32);
    if (g == 0) lred[wave][i16] = sum;
    __syncthreads();
    l = l * keep + ((lred[0][i16] + lred[1][i16]) + (lred[2][i16] + lred[3][i16]));
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[j][r] *= keep;
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      const u32x2 plo = *(const u32x2*)&pl[i16][32 * kk + 4 * g], phi = *(const u32x2*)&pl[i16][32 * kk + 16 + 4 * g];
      const u32x4 pb = {plo.x, plo.y, phi.x, phi.y};
#pragma unroll
      for (int j = 0; j < NT; ++j) {
        const int col = 16 * (wave + 4 * j);
        if (col < p.kv_rank) {  // uniform; a last tile may reach into the rotated part: never stored
          const u32x2 a0 = lds_read_tr16(&cl[(32 * kk + 4 * g + (i16 >> 2)) * pitch + col + 4 * (i16 & 3)]);
          const u32x2 a1 = lds_read_tr16(&cl[(32 * kk + 16 + 4 * g + (i16 >> 2)) * pitch + col + 4 * (i16 & 3)]);
          acc[j] = mfma16x16x32<T>(u32x4{a0.x, a0.y, a1.x, a1.y}, pb, acc[j]);
        }
      }
    }
  }
  if (h0 + i16 < p.heads) {
    float* dst = p.part + (((long)tok * p.heads + h0 + i16) * p.splits + split) * (p.kv_rank + 2);
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int c = 16 * (wave + 4 * j) + 4 * g + r;
        if (c < p.kv_rank) dst[c] = acc[j][r];
      }
    if (wave == 0 && g == 0) {
      dst[p.kv_rank] = m;
      dst[p.kv_rank + 1] = l;
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
  const long stride = p.kv_rank + 2;
  const float* part = p.part + ((long)tok * p.heads + h) * p.splits * stride;
  if (t < kWave) {  // the splits' shares, one per lane
    const bool in = t < p.splits;
    const float mm = in ? part[t * stride + p.kv_rank] : -1e30f, ll = in ? part[t * stride + p.kv_rank + 1] : 0.f;
    const float e = exp2f(mm - wave_max(mm));
    const float l = wave_sum(e * ll);
    if (in) ws[t] = ll > 0.f ? e / l : 0.f;
  }
  __syncthreads();
  for (int r = t; r < p.kv_rank; r += 256) {
    float a = 0.f;
#pragma unroll 8
    for (int s = 0; s < p.splits; ++s) a = fmaf(ws[s], part[s * stride + r], a);
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
// prefill: grid (heads, tiles of 32 NW queries, longest first) of one batch row; NW waves of 32 queries,
// two LDS stages of 64 keys: the next block's loads are in flight while one is attended to
// ---------------------------------------------------------------------------------------
template <typename T, int DKC, int DVT, int NW>
__global__ void __launch_bounds__(64 * NW, NW == 8 ? 2 : 1) latent_prefill_kernel(const LatentParams p) {
  constexpr int KPITCH = DKC * 32 + 8, VPITCH = DVT * 16 + 16;  // elements per LDS row
  constexpr int THREADS = 64 * NW, QT = 32 * NW;
  constexpr int KCH = 64 * DKC * 4, VCH = 64 * DVT * 2;  // 16-byte chunks per block
  constexpr int KI = (KCH + THREADS - 1) / THREADS, VI = (VCH + THREADS - 1) / THREADS;
  constexpr int STAGE = 64 * (KPITCH + VPITCH);
  uint16_t* smem = (uint16_t*)la_smem;  // first the queries, [QT][KPITCH], then two stages of K | V rows
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, g = lane >> 4, i16 = lane & 15;
  const int h = blockIdx.x, qt0 = ((int)gridDim.y - 1 - (int)blockIdx.y) * QT;
  const int hd = p.dim + p.rot, dk = hd;
  const long first_row = p.row_start ? p.row_start[p.b0] : 0;
  // queries: rotated, rounded, through LDS into operand registers (column i16, k-chunk g)
  for (int c = t; c < QT * DKC * 4; c += THREADS) {
    const int r = c / (DKC * 4), e0 = (c - r * DKC * 4) * 8;
    uint16_t v[8];
    const int tq = qt0 + r;
    const long tok = (long)p.b0 * p.t + (tq < p.t ? tq : p.t - 1);
    const uint16_t* qh = (const uint16_t*)p.q + (tok * p.heads + h) * hd;
#pragma unroll
    for (int j = 0; j < 8; ++j)
      v[j] = e0 + j < dk ? T::pack(rotated_q<T>(qh, p.cos_sin + tok * p.rot, p.dim, p.rot, e0 + j)) : (uint16_t)0;
    *(u32x4*)&smem[r * KPITCH + e0] = u32x4{(uint32_t)v[0] | ((uint32_t)v[1] << 16), (uint32_t)v[2] | ((uint32_t)v[3] << 16),
                                            (uint32_t)v[4] | ((uint32_t)v[5] << 16), (uint32_t)v[6] | ((uint32_t)v[7] << 16)};
  }
  __syncthreads();
  u32x4 q[2][DKC];
#pragma unroll
  for (int qt = 0; qt < 2; ++qt)
#pragma unroll
    for (int c = 0; c < DKC; ++c) q[qt][c] = *(const u32x4*)&smem[(wave * 32 + qt * 16 + i16) * KPITCH + c * 32 + 8 * g];
  __syncthreads();
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
  const bool v8 = p.dim % 8 == 0 && p.rot % 8 == 0 && p.vdim % 8 == 0;  // 16-byte chunks stay aligned
  const u32x4 zero = {0u, 0u, 0u, 0u};
  u32x4 rk[KI], rv[VI];
  auto fetch = [&](int s0) {
    if (v8) {
#pragma unroll
      for (int i = 0; i < KI; ++i) {
        const int c = t + THREADS * i, r = c / (DKC * 4), e0 = (c - r * DKC * 4) * 8;
        const long row = s0 + r < n_keys ? s0 + r : n_keys - 1;
        const uint16_t* src = e0 < p.dim ? kbase + row * kvp + e0 : rc + row * p.rot + (e0 < dk ? e0 - p.dim : 0);
        rk[i] = ld16(src);
        rk[i] = e0 < dk ? rk[i] : zero;
      }
#pragma unroll
      for (int i = 0; i < VI; ++i) {
        const int c = t + THREADS * i, r = c / (DVT * 2), e0 = (c - r * DVT * 2) * 8;
        const long row = s0 + r < n_keys ? s0 + r : n_keys - 1;
        rv[i] = ld16(vbase + row * kvp + (e0 < p.vdim ? e0 : 0));
        rv[i] = e0 < p.vdim ? rv[i] : zero;
      }
    }
  };
  auto put = [&](int s0, int buf) {
    uint16_t *kl = smem + buf * STAGE, *vl = kl + 64 * KPITCH;
    if (v8) {
#pragma unroll
      for (int i = 0; i < KI; ++i) {
        const int c = t + THREADS * i, r = c / (DKC * 4), e0 = (c - r * DKC * 4) * 8;
        if (KCH % THREADS == 0 || c < KCH) *(u32x4*)&kl[r * KPITCH + e0] = rk[i];
      }
#pragma unroll
      for (int i = 0; i < VI; ++i) {
        const int c = t + THREADS * i, r = c / (DVT * 2), e0 = (c - r * DVT * 2) * 8;
        if (VCH % THREADS == 0 || c < VCH) *(u32x4*)&vl[r * VPITCH + e0] = rv[i];
      }
    } else {  // rows whose parts are no multiples of 16 bytes: element by element
      for (int c = t; c < 64 * DKC * 32; c += THREADS) {
        const int r = c / (DKC * 32), e = c - r * DKC * 32;
        const long row = s0 + r < n_keys ? s0 + r : n_keys - 1;
        kl[r * KPITCH + e] = e < p.dim ? kbase[row * kvp + e] : (e < dk ? rc[row * p.rot + e - p.dim] : (uint16_t)0);
      }
      for (int c = t; c < 64 * DVT * 16; c += THREADS) {
        const int r = c / (DVT * 16), e = c - r * DVT * 16;
        const long row = s0 + r < n_keys ? s0 + r : n_keys - 1;
        vl[r * VPITCH + e] = e < p.vdim ? vbase[row * kvp + e] : (uint16_t)0;
      }
    }
  };
  // this wave's queries, as positions counted from lo
  const int wq0 = (int)((long)p.q_first + qt0 + wave * 32 - lo), wq1 = wq0 + 31;
  auto attend = [&](int s0, int buf) {
    const uint16_t *kl = smem + buf * STAGE, *vl = kl + 64 * KPITCH;
    f32x4 s4[2][4];
#pragma unroll
    for (int kt = 0; kt < 4; ++kt) {
#pragma unroll
      for (int qt = 0; qt < 2; ++qt) s4[qt][kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int c = 0; c < DKC; ++c) {
        const u32x4 a = *(const u32x4*)&kl[(kt * 16 + i16) * KPITCH + c * 32 + 8 * g];
#pragma unroll
        for (int qt = 0; qt < 2; ++qt) s4[qt][kt] = mfma16x16x32<T>(a, q[qt][c], s4[qt][kt]);
      }
    }
    const bool full = s0 + 63 <= wq0 && (p.window <= 0 || s0 >= wq1 - p.window + 1);
    u32x4 pb[2][2];
#pragma unroll
    for (int qt = 0; qt < 2; ++qt) {
      const int qp = wq0 + qt * 16 + i16;
      float mx = -INFINITY;
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          float v = s4[qt][kt][r] * sc;
          if (!full) {
            const int s = s0 + kt * 16 + 4 * g + r;
            if (s > qp || (p.window > 0 && s <= qp - p.window)) v = -INFINITY;
          }
          s4[qt][kt][r] = v;
          mx = fmaxf(mx, v);
        }
      mx = fmaxf(mx, __shfl_xor(mx, 16));
      mx = fmaxf(mx, __shfl_xor(mx, 32));
      if (__any(mx > m[qt])) {
        const float mn = fmaxf(m[qt], mx), keep = exp2f(m[qt] - mn);
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
        for (int r = 0; r < 4; ++r) { e[kt][r] = exp2f(s4[qt][kt][r] - m[qt]); sum += e[kt][r]; }
      l[qt] += sum;  // this lane's keys only; the lane groups are added up at the end
#pragma unroll
      for (int kk = 0; kk < 2; ++kk)
        pb[qt][kk] = u32x4{T::pack2(e[2 * kk][0], e[2 * kk][1]), T::pack2(e[2 * kk][2], e[2 * kk][3]),
                           T::pack2(e[2 * kk + 1][0], e[2 * kk + 1][1]), T::pack2(e[2 * kk + 1][2], e[2 * kk + 1][3])};
    }
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int j = 0; j < DVT; ++j) {
        const u32x2 a0 = lds_read_tr16(&vl[(32 * kk + 4 * g + (i16 >> 2)) * VPITCH + 16 * j + 4 * (i16 & 3)]);
        const u32x2 a1 = lds_read_tr16(&vl[(32 * kk + 16 + 4 * g + (i16 >> 2)) * VPITCH + 16 * j + 4 * (i16 & 3)]);
        const u32x4 va = {a0.x, a0.y, a1.x, a1.y};
#pragma unroll
        for (int qt = 0; qt < 2; ++qt) acc[qt][j] = mfma16x16x32<T>(va, pb[qt][kk], acc[qt][j]);
      }
  };
  if (n_keys > 0) {
    fetch(0);
    put(0, 0);
  }
  for (int s0 = 0, buf = 0; s0 < n_keys; s0 += 64, buf ^= 1) {
    __syncthreads();  // block s0 is in its stage; everybody is done with the other one
    const bool more = s0 + 64 < n_keys;
    if (more) fetch(s0 + 64);
    // (blocks that none of the wave's queries sees are skipped)
    if (s0 <= wq1 && (p.window <= 0 || s0 + 63 > wq0 - p.window)) attend(s0, buf);
    if (more) put(s0 + 64, buf ^ 1);
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

template <typename T>
static int launch_latent_decode(hipStream_t s, const LatentParams& p) {
  const int tokens = p.batch * p.t;
  if (tokens > 65535 || p.kv_rank > 1024) return MUI_ERR_UNSUPPORTED;
  hipLaunchKernelGGL((latent_absorb_kernel<T>), dim3(p.heads, ceil_div(p.kv_rank, 64), ceil_div(tokens, kAbsTok)),
                     dim3(256), 0, s, p);
  const dim3 grid(p.splits, ceil_div(p.heads, 16), tokens);
  const size_t lds = (size_t)80 * (p.kp + 8) * 2;
  int st;
  if (p.kv_rank <= 128) st = launch_with_lds(latent_decode_kernel<T, 2>, grid, dim3(256), lds, s, p);
  else if (p.kv_rank <= 256) st = launch_with_lds(latent_decode_kernel<T, 4>, grid, dim3(256), lds, s, p);
  else if (p.kv_rank <= 512) st = launch_with_lds(latent_decode_kernel<T, 8>, grid, dim3(256), lds, s, p);
  else st = launch_with_lds(latent_decode_kernel<T, 16>, grid, dim3(256), lds, s, p);
  if (st != MUI_OK) return st;
  return launch_with_lds(latent_output_kernel<T>, dim3(p.heads, ceil_div(p.vdim, 32), tokens), dim3(256),
                         (size_t)p.kv_rank * 4, s, p);
}

template <typename T, int DKC, int DVT, int NW>
static int launch_latent_prefill_w(hipStream_t s, const LatentParams& p) {
  constexpr size_t kv = (size_t)2 * 64 * (DKC * 32 + 8 + DVT * 16 + 16) * 2, q = (size_t)32 * NW * (DKC * 32 + 8) * 2;
  const int tiles = ceil_div(p.t, 32 * NW);
  if (tiles > 65535) return MUI_ERR_UNSUPPORTED;
  return launch_with_lds(latent_prefill_kernel<T, DKC, DVT, NW>, dim3(p.heads, tiles), dim3(64 * NW), kv > q ? kv : q, s, p);
}

template <typename T, int DKC, int DVT>
static int launch_latent_prefill_t(hipStream_t s, const LatentParams& p) {
  // 256 queries per workgroup once that leaves most of the chip something to do
  if (p.heads * ceil_div(p.t, 256) * 2 >= device_cus()) return launch_latent_prefill_w<T, DKC, DVT, 8>(s, p);
  return launch_latent_prefill_w<T, DKC, DVT, 4>(s, p);
}

static bool prefill_covers(int dk, int vdim) { return dk <= 256 && vdim <= 256; }

template <typename T>
static int launch_latent_prefill(hipStream_t s, const LatentParams& p) {
  const int dk = p.dim + p.rot;
  if (dk <= 64 && p.vdim <= 64) return launch_latent_prefill_t<T, 2, 4>(s, p);
  if (dk <= 96 && p.vdim <= 64) return launch_latent_prefill_t<T, 3, 4>(s, p);
  if (dk <= 128 && p.vdim <= 128) return launch_latent_prefill_t<T, 4, 8>(s, p);
  if (dk <= 192 && p.vdim <= 128) return launch_latent_prefill_t<T, 6, 8>(s, p);
  if (prefill_covers(dk, p.vdim)) return launch_latent_prefill_w<T, 8, 16, 4>(s, p);
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

static int latent_kp(int kv_rank, int rot_dim) { return (kv_rank + rot_dim + 31) / 32 * 32; }

// keys per split and number of splits of the decode kernel for spans of up to `span` keys
static void latent_split(int batch, int t, int heads, int span, int* splits, int* split_keys) {
  const int groups = batch * t * ceil_div(heads, 16);
  int want = device_cus() * 2 / (groups > 0 ? groups : 1);
  want = want < 1 ? 1 : (want > kMaxSplits ? kMaxSplits : want);
  const int blocks = ceil_div(span, 64);
  int per = ceil_div(blocks, want);
  if (per < 2 && blocks > 8) per = 2;  // merging costs a split's partial result per head
  *split_keys = per * 64;
  *splits = ceil_div(blocks, per);
}

extern "C" int mui_latent_attention_route(int dtype, int tokens, int heads, int dim, int rot_dim, int vdim, int kv_rank) {
  if (dtype == MUI_DTYPE_F32 || kv_rank % 8) return MUI_LATENT_PLAIN;
  if (tokens > MUI_MAX_TOKENS && prefill_covers(dim + rot_dim, vdim)) return MUI_LATENT_PREFILL;
  return kv_rank <= 1024 && (size_t)80 * (latent_kp(kv_rank, rot_dim) + 8) * 2 <= 150 * 1024 ? MUI_LATENT_DECODE
                                                                                             : MUI_LATENT_PLAIN;
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
  if (kv_rank % 8) return MUI_ERR_UNSUPPORTED;
  if (!aligned16(w_uk) || !aligned16(w_uv) || !aligned16(c_cache) || !aligned16(r_cache) || c_batch_stride % 8 ||
      (rot_dim % 8 == 0 && r_batch_stride % 8) || ((uintptr_t)scratch & 255))
    return MUI_ERR_ALIGNMENT;
  p.kp = latent_kp(kv_rank, rot_dim);
  latent_split(batch, t, heads, span, &p.splits, &p.split_keys);
  p.q_abs = scratch;
  p.part = (float*)((char*)scratch + ((size_t)batch * t * heads * p.kp * 2 + 255) / 256 * 256);
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
