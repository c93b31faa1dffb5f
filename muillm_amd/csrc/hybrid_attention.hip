// Grouped-query attention of hybrid decoders, over key and value rows cached per token:
//   score[h, s] = (q_h . k_s) * scale, capped as softcap * tanh(score / softcap) where softcap > 0
//   out[h] = sigmoid(gate_h) * sum_s softmax(score)_s v_s
// A query at position i sees position j <= i where i - j < window, or j < keep_first (sinks: the first tokens
// of the sequence stay visible), or everything with window 0. Key and value sizes may differ.
//
//   prepare   from the projections' output q | k | v: RMS norm over ALL rows of q (and of k), rotation of the
//             first `rot` dimensions of every head (pairs 2 i, 2 i + 1), k and v into the caches
//   decode    (few tokens) the query heads of a KV head are the columns of the matrix instructions, the key
//             range is split over workgroups; combine merges the splits and applies the gate
//   prefill   (prompts) a flash kernel: 32 queries per wave, 64 keys per step, K double-buffered; the waves of a
//             workgroup are query heads of one KV head where there are several, else blocks of queries
//   plain     one workgroup per query and head: fp32 models, sizes the others do not cover.
//
// Visible keys are counted compactly: n = 0 .. kf - 1 are the kept first tokens in front of the window, n >= kf
// continue at the window's start, so kept tokens cost a walk over the window no special case but a shift.
// Positions: a token's slot in the cache minus its row's first slot (left-padded batches).
#include "hybrid.cuh"

namespace mui {

struct HybridAttnParams {
  const void* proj;      // [tokens, pitch]: q | k | v at the offsets below
  long pitch, k_off, v_off;
  const void *q_gain, *k_gain;  // [heads * dim], [kv_heads * dim], or null: no norm
  float eps;
  const double* inv_freq;  // [rot / 2]
  int rot;
  void* q_out;  // [tokens, heads * dim]

  const void* q;           // [tokens, heads * dim], normed and rotated
  void *k_cache, *v_cache; // [batch, max_cache_len, kv_heads * dim | kv_heads * vdim]
  long k_batch, v_batch;
  const void* gate;        // [tokens, gate_pitch], heads * vdim of it; or null
  long gate_pitch;
  const int64_t* cache_position;  // [t], consecutive slots
  const int64_t* row_start;       // [batch] or null
  int batch, t, heads, kv_heads, dim, vdim, window, keep, max_cache_len;
  float scale, softcap;
  void* out;  // [tokens, heads * vdim]

  float *part, *part_ml;  // decode: [tokens, heads, splits, vdim], [tokens, heads, splits, 2]
  int splits, split_keys;
  int head_waves;  // prefill: query heads per workgroup
};

// ---------------------------------------------------------------------------------------
// prepare: one workgroup per token
// ---------------------------------------------------------------------------------------
extern __shared__ __align__(16) unsigned char ha_smem[];
struct CosSin { float c, s; };

template <typename T, bool VEC>
__global__ void __launch_bounds__(512) hybrid_prepare_kernel(const HybridAttnParams p) {
  typedef typename T::storage S;
  __shared__ float red[2][8];
  CosSin* cs = (CosSin*)ha_smem;  // dim / 2 (cos, sin); (1, 0) behind the rotated dimensions
  const int tok = blockIdx.x, b = tok / p.t, t = threadIdx.x, nt = blockDim.x;
  const S* row = (const S*)p.proj + (long)tok * p.pitch;
  const S *qr = row, *kr = row + p.k_off, *vr = row + p.v_off;
  const int nq = p.heads * p.dim, nk = p.kv_heads * p.dim, nv = p.kv_heads * p.vdim;
  const long slot = p.cache_position[tok - b * p.t];
  const long pos = slot - (p.row_start ? p.row_start[b] : 0);
  for (int i = t; i < (p.dim + 1) / 2; i += nt) {
    float c = 1.f, s = 0.f;
    if (2 * i < p.rot) rope_angle((double)(pos > 0 ? pos : 0), p.inv_freq[i], c, s);
    cs[i] = CosSin{c, s};
  }
  float sq = 0.f, sk = 0.f;
  auto squares = [&](const S* x, int n) {
    float a = 0.f;
    if constexpr (VEC) {
#pragma unroll 2
      for (int c = t * 8; c < n; c += nt * 8) {
        float f[8];
        load8<T>(x + c, f);
#pragma unroll
        for (int i = 0; i < 8; ++i) a = fmaf(f[i], f[i], a);
      }
    } else {
      for (int c = t; c < n; c += nt) {
        const float f = T::one(x[c]);
        a = fmaf(f, f, a);
      }
    }
    return wave_sum(a);
  };
  if (p.q_gain) sq = squares(qr, nq);
  if (p.k_gain) sk = squares(kr, nk);
  if ((t & 63) == 0) {
    red[0][t >> 6] = sq;
    red[1][t >> 6] = sk;
  }
  __syncthreads();
  sq = sk = 0.f;
  for (int w = 0; w < nt / 64; ++w) {
    sq += red[0][w];
    sk += red[1][w];
  }
  const float rq = p.q_gain ? rsqrtf(sq / (float)nq + p.eps) : 1.f, rk = p.k_gain ? rsqrtf(sk / (float)nk + p.eps) : 1.f;
  auto emit = [&](const S* x, const S* gain, float rs, int n, S* dst) {
    if constexpr (VEC) {
#pragma unroll 2
      for (int c = t * 8; c < n; c += nt * 8) {
        float f[8], g[8];
        load8<T>(x + c, f);
        if (gain) {
          load8<T>(gain + c, g);
#pragma unroll
          for (int i = 0; i < 8; ++i) f[i] = g[i] * (f[i] * rs);
        }
        const int e = (c % p.dim) >> 1;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float co = cs[e + i].c, si = cs[e + i].s, u = f[2 * i], v = f[2 * i + 1];
          g[2 * i] = u * co - v * si;
          g[2 * i + 1] = v * co + u * si;
        }
        store8<T>(dst + c, g);
      }
    } else {
      for (int c = t; c < n; c += nt) {
        const int e = c % p.dim;
        auto at = [&](int i) { return gain ? T::one(gain[i]) * (T::one(x[i]) * rs) : T::one(x[i]); };
        float y = at(c);
        if (e < p.rot) {
          const float co = cs[e >> 1].c, si = cs[e >> 1].s;
          const float o = at(e & 1 ? c - 1 : c + 1);
          y = e & 1 ? y * co + o * si : y * co - o * si;
        }
        dst[c] = T::pack(y);
      }
    }
  };
  emit(qr, (const S*)p.q_gain, rq, nq, (S*)p.q_out + (long)tok * nq);
  if (slot < 0 || slot >= p.max_cache_len) return;
  emit(kr, (const S*)p.k_gain, rk, nk, (S*)p.k_cache + b * p.k_batch + slot * nk);
  S* vd = (S*)p.v_cache + b * p.v_batch + slot * nv;
  if constexpr (VEC) {
    for (int c = t * 8; c < nv; c += nt * 8) {
      float f[8];
      load8<T>(vr + c, f);
      store8<T>(vd + c, f);
    }
  } else {
    for (int c = t; c < nv; c += nt) vd[c] = vr[c];
  }
}

// ---------------------------------------------------------------------------------------
// visible keys of the queries in slots lo_slot .. hi_slot of batch row b, counted compactly
// ---------------------------------------------------------------------------------------
struct KeyRange {
  long first;   // slot of position 0
  int kf, n;    // kept tokens in front of the window, keys in all
  int shift;    // position of key n >= kf: n + shift
  __device__ __forceinline__ long slot(int i) const { return first + (i < kf ? i : i + shift); }
};

__device__ __forceinline__ KeyRange key_range(const HybridAttnParams& p, int b, long lo_slot, long hi_slot) {
  KeyRange r;
  r.first = p.row_start ? p.row_start[b] : 0;
  r.first = r.first > 0 ? r.first : 0;
  const long hi = hi_slot < p.max_cache_len ? hi_slot : p.max_cache_len - 1;
  long lo = p.window > 0 ? lo_slot - p.window + 1 : r.first;
  lo = lo > r.first ? lo : r.first;
  const long gap = lo - r.first;
  r.kf = (int)(p.keep < gap ? p.keep : gap);
  r.shift = (int)(gap - r.kf);
  r.n = hi >= lo ? r.kf + (int)(hi - lo + 1) : 0;
  return r;
}

__device__ __forceinline__ float sigmoid_f32(float x) { return 1.f / (1.f + expf(-x)); }

// ---------------------------------------------------------------------------------------
// plain: grid (heads, tokens)
// ---------------------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256) hybrid_plain_kernel(const HybridAttnParams p) {
  typedef typename T::storage S;
  __shared__ float red[4], pr[256];
  float* q = (float*)ha_smem;  // dim
  float* o = q + p.dim;        // vdim
  const int h = blockIdx.x, tok = blockIdx.y, b = tok / p.t, t = threadIdx.x;
  const int kvh = h / (p.heads / p.kv_heads);
  const S* qh = (const S*)p.q + ((long)tok * p.heads + h) * p.dim;
  for (int i = t; i < p.dim; i += 256) q[i] = T::one(qh[i]);
  for (int i = t; i < p.vdim; i += 256) o[i] = 0.f;
  __syncthreads();
  const long slot = p.cache_position[tok - b * p.t];
  const KeyRange kr = key_range(p, b, slot, slot);
  const long kp = (long)p.kv_heads * p.dim, vp = (long)p.kv_heads * p.vdim;
  const S* kc = (const S*)p.k_cache + b * p.k_batch + (long)kvh * p.dim;
  const S* vc = (const S*)p.v_cache + b * p.v_batch + (long)kvh * p.vdim;
  float m = -1e30f, l = 0.f;
  for (int s0 = 0; s0 < kr.n; s0 += 256) {
    float sc = -INFINITY;
    if (s0 + t < kr.n) {
      const S* k = kc + kr.slot(s0 + t) * kp;
      float a = 0.f;
      for (int d = 0; d < p.dim; ++d) a = fmaf(q[d], T::one(k[d]), a);
      sc = a * p.scale;
      if (p.softcap > 0.f) sc = p.softcap * tanhf(sc / p.softcap);
    }
    float mx = wave_max(sc);
    __syncthreads();
    if ((t & 63) == 0) red[t >> 6] = mx;
    __syncthreads();
    mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float mn = fmaxf(m, mx), keep = expf(m - mn), e = expf(sc - mn);
    pr[t] = e;
    l = l * keep + block_sum256(e, red);  // (barriers: pr is complete)
    m = mn;
    const int n = kr.n - s0 < 256 ? kr.n - s0 : 256;
    for (int v = t; v < p.vdim; v += 256) {
      float a = o[v] * keep;
      for (int j = 0; j < n; ++j) a = fmaf(pr[j], T::one(vc[kr.slot(s0 + j) * vp + v]), a);
      o[v] = a;
    }
    __syncthreads();
  }
  const float inv = l > 0.f ? 1.f / l : 0.f;
  for (int v = t; v < p.vdim; v += 256) {
    float y = o[v] * inv;
    if (p.gate) y *= sigmoid_f32(T::one(((const S*)p.gate)[tok * p.gate_pitch + (long)h * p.vdim + v]));
    ((S*)p.out)[((long)tok * p.heads + h) * p.vdim + v] = T::pack(y);
  }
}

// a score in units of log 2: scale, or scale and cap (c1 = 2 scale log2(e) / cap, c2 = cap log2(e):
// cap tanh(x) = cap - 2 cap / (e^{2x} + 1))
template <bool CAP>
__device__ __forceinline__ float score_log2(float s, float c1, float c2) {
  if constexpr (!CAP) return s * c1;
  return fmaf(-2.f * c2, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s * c1) + 1.f), c2);
}

constexpr float kLog2eF = 1.4426950408889634f;

// ---------------------------------------------------------------------------------------
// decode: grid (splits, kv_heads * groups of 16 query heads, tokens); four waves, 64 keys per block
//   scores: wave w takes keys 16 w ..: A = key rows, B = the heads' queries; lane (g, i) ends up with head i,
//           keys 16 w + 4 g + r
//   values: O^T[v, head] += V^T P^T, the value rows read back transposed; wave w owns value tiles w, w + 4, ..
// ---------------------------------------------------------------------------------------
constexpr int kHdKeys = 64;
constexpr int kHdMaxSplits = 64;

__device__ __forceinline__ int hybrid_live_splits(const HybridAttnParams& p, const KeyRange& kr) {
  return (kr.n + p.split_keys - 1) / p.split_keys;
}

template <typename T, int DKC, int DVT, bool CAP>  // dim <= 32 DKC, vdim <= 16 DVT
__global__ void __launch_bounds__(256) hybrid_decode_kernel(const HybridAttnParams p) {
  constexpr int KG = DKC / 2, VG = DVT / 4, NV = DVT / 4;
  __shared__ float mred[4][16], lred[4][16];
  __shared__ __align__(16) uint16_t pl[16][kHdKeys + 8];
  uint16_t* kl = (uint16_t*)ha_smem;       // [KG][64][64]
  uint16_t* vl = kl + KG * kHdKeys * 64;   // [VG][64][64]
  const int t = threadIdx.x, lane = t & 63, wave = __builtin_amdgcn_readfirstlane(t >> 6), g = lane >> 4, i16 = lane & 15;
  const int share = p.heads / p.kv_heads, groups = (share + 15) / 16;
  const int split = blockIdx.x, kvh = blockIdx.y / groups, hg = (blockIdx.y - kvh * groups) * 16, tok = blockIdx.z, b = tok / p.t;
  const long slot = p.cache_position[tok - b * p.t];
  const KeyRange kr = key_range(p, b, slot, slot);
  if (split >= hybrid_live_splits(p, kr) && p.splits > 1) return;  // uniform for the workgroup
  const int s_begin = split * p.split_keys;
  const int s_end = s_begin + p.split_keys < kr.n ? s_begin + p.split_keys : kr.n;
  const long kp = (long)p.kv_heads * p.dim, vp = (long)p.kv_heads * p.vdim;
  const uint16_t* kc = (const uint16_t*)p.k_cache + b * p.k_batch + (long)kvh * p.dim;
  const uint16_t* vc = (const uint16_t*)p.v_cache + b * p.v_batch + (long)kvh * p.vdim;
  const int hh = kvh * share + (hg + i16 < share ? hg + i16 : share - 1);  // this lane's head (columns past the share repeat one)
  u32x4 q[DKC];
#pragma unroll
  for (int c = 0; c < DKC; ++c) {
    const int e = c * 32 + 8 * g;
    const u32x4 v = ld16((const uint16_t*)p.q + ((long)tok * p.heads + hh) * p.dim + (e < p.dim ? e : 0));
    q[c] = e < p.dim ? v : u32x4{0u, 0u, 0u, 0u};
  }
  f32x4 acc[NV];
#pragma unroll
  for (int j = 0; j < NV; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -1e30f, l = 0.f;
  const float c1 = CAP ? 2.f * p.scale / p.softcap * kLog2eF : p.scale * kLog2eF, c2 = p.softcap * kLog2eF;
  const int lrow = wave * 8 + (lane >> 3), lc = ((lane & 7) ^ tile_swz(lrow)) * 8;
  for (int s0 = s_begin; s0 < s_end; s0 += kHdKeys) {
    __syncthreads();  // the previous block is done with
    // rows past the split repeat its last one (masked), columns past a row's end repeat its start (the queries
    // hold zeros there; such values are never stored)
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int n = s0 + lrow + 32 * u;
      const long s = kr.slot(n < s_end ? n : s_end - 1);
#pragma unroll
      for (int cg = 0; cg < KG; ++cg)
        load_lds16(kc + s * kp + (cg * 64 + lc < p.dim ? cg * 64 + lc : 0), &kl[(cg * 64 + wave * 8 + 32 * u) * 64]);
    }
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int n = s0 + lrow + 32 * u;
      const long s = kr.slot(n < s_end ? n : s_end - 1);
#pragma unroll
      for (int cg = 0; cg < VG; ++cg)
        load_lds16(vc + s * vp + (cg * 64 + lc < p.vdim ? cg * 64 + lc : 0), &vl[(cg * 64 + wave * 8 + 32 * u) * 64]);
    }
    wait_loads<2 * VG>();  // the keys
    __syncthreads();
    f32x4 s4 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < DKC; ++c) s4 = mfma16x16x32<T>(*(const u32x4*)&kl[tile_at<kHdKeys>(16 * wave + i16, c * 32 + 8 * g)], q[c], s4);
    float mx = -INFINITY;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      s4[r] = s0 + 16 * wave + 4 * g + r < s_end ? score_log2<CAP>(s4[r], c1, c2) : -INFINITY;
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
    wait_loads<0>();  // the values
    __syncthreads();
    l = l * keep + ((lred[0][i16] + lred[1][i16]) + (lred[2][i16] + lred[3][i16]));
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[j][r] *= keep;
#pragma unroll
    for (int kk = 0; kk < kHdKeys / 32; ++kk) {
      const u32x2 plo = *(const u32x2*)&pl[i16][32 * kk + 4 * g], phi = *(const u32x2*)&pl[i16][32 * kk + 16 + 4 * g];
      const u32x4 pb = {plo.x, plo.y, phi.x, phi.y};
      const int row = 32 * kk + 4 * g + (i16 >> 2);
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const int col = 16 * (wave + 4 * j) + 4 * (i16 & 3);
        const u32x2 a0 = lds_read_tr16(&vl[tile_at<kHdKeys>(row, col)]), a1 = lds_read_tr16(&vl[tile_at<kHdKeys>(row + 16, col)]);
        acc[j] = mfma16x16x32<T>(u32x4{a0.x, a0.y, a1.x, a1.y}, pb, acc[j]);
      }
    }
  }
  if (hg + i16 >= share) return;
  if (p.splits == 1) {
    const float inv = l > 0.f ? 1.f / l : 0.f;
    const uint16_t* gr = (const uint16_t*)p.gate + tok * p.gate_pitch + (long)hh * p.vdim;
    uint16_t* dst = (uint16_t*)p.out + ((long)tok * p.heads + hh) * p.vdim;
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int v = 16 * (wave + 4 * j) + 4 * g + r;
        if (v < p.vdim) dst[v] = T::pack(acc[j][r] * inv * (p.gate ? sigmoid_f32(T::one(gr[v])) : 1.f));
      }
    return;
  }
  const long at = ((long)tok * p.heads + hh) * p.splits + split;
#pragma unroll
  for (int j = 0; j < NV; ++j) {
    const int v = 16 * (wave + 4 * j) + 4 * g;  // (vdim is a multiple of 8)
    if (v < p.vdim) *(f32x4*)&p.part[at * p.vdim + v] = acc[j];
  }
  if (wave == 0 && g == 0) {
    p.part_ml[at * 2] = m;
    p.part_ml[at * 2 + 1] = l;
  }
}

// grid (heads, tokens): merges the splits of a head, gate, rounding
template <typename T>
__global__ void __launch_bounds__(128) hybrid_combine_kernel(const HybridAttnParams p) {
  __shared__ float ws[kHdMaxSplits];
  const int h = blockIdx.x, tok = blockIdx.y, b = tok / p.t, t = threadIdx.x;
  const long at = ((long)tok * p.heads + h) * p.splits;
  const float* part = p.part + at * p.vdim;
  const long slot = p.cache_position[tok - b * p.t];
  const int live = hybrid_live_splits(p, key_range(p, b, slot, slot));
  if (t < kWave) {  // the splits' shares, one per lane
    const bool in = t < live;
    const float mm = in ? p.part_ml[(at + t) * 2] : -1e30f, ll = in ? p.part_ml[(at + t) * 2 + 1] : 0.f;
    const float e = exp2f(mm - wave_max(mm));
    const float all = wave_sum(e * ll);
    ws[t] = in ? e / all : 0.f;
  }
  __syncthreads();
  for (int v = t; v < p.vdim; v += 128) {
    float a = 0.f;
    for (int s0 = 0; s0 < live; s0 += 16) {  // splits past the live ones repeat the last one with a share of zero
      float x[16];
#pragma unroll
      for (int u = 0; u < 16; ++u) x[u] = part[(long)(s0 + u < live ? s0 + u : live - 1) * p.vdim + v];
#pragma unroll
      for (int u = 0; u < 16; ++u) a = fmaf(ws[s0 + u], x[u], a);
    }
    if (p.gate) a *= sigmoid_f32(T::one(((const uint16_t*)p.gate)[tok * p.gate_pitch + (long)h * p.vdim + v]));
    ((uint16_t*)p.out)[((long)tok * p.heads + h) * p.vdim + v] = T::pack(a);
  }
}

// ---------------------------------------------------------------------------------------
// prefill: grid (batch * heads / head_waves, tiles of queries, longest first); NW waves, wave w serves query head
// w % head_waves and the block of 32 queries w / head_waves. LDS holds two stages of 64 keys and one of their
// values: while block s is multiplied with the queries, its values and the keys of block s + 1 are on their way.
// ---------------------------------------------------------------------------------------
template <int DKC, int DVT>
constexpr size_t hybrid_prefill_lds() { return (size_t)64 * (2 * DKC * 32 + DVT * 16) * 2; }

template <typename T, int DKC, int DVT, int NW, bool CAP>
__global__ void __launch_bounds__(64 * NW, DKC > 4 ? 1 : 2) hybrid_prefill_kernel(const HybridAttnParams p) {
  static_assert(DKC % 2 == 0 && DVT % 4 == 0 && (NW == 2 || NW == 4), "tiles of 64 columns");
  constexpr int KG = DKC / 2, VG = DVT / 4, RB = 8 / NW, RSTEP = 8 * NW, KSTAGE = KG * 64 * 64;
  uint16_t* smem = (uint16_t*)ha_smem;
  uint16_t* vl = smem + 2 * KSTAGE;
  const int t = threadIdx.x, lane = t & 63, wave = __builtin_amdgcn_readfirstlane(t >> 6), g = lane >> 4, i16 = lane & 15;
  const int hw = p.head_waves, hgs = p.heads / hw, b = blockIdx.x / hgs;
  const int h = (blockIdx.x - b * hgs) * hw + wave % hw, kvh = h / (p.heads / p.kv_heads);
  const int QT = 32 * (NW / hw), qt0 = ((int)gridDim.y - 1 - (int)blockIdx.y) * QT, wq = qt0 + 32 * (wave / hw);
  f32x4 acc[2][DVT];
  float m[2] = {-1e30f, -1e30f}, l[2] = {0.f, 0.f};
#pragma unroll
  for (int qt = 0; qt < 2; ++qt)
#pragma unroll
    for (int j = 0; j < DVT; ++j) acc[qt][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const float c1 = CAP ? 2.f * p.scale / p.softcap * kLog2eF : p.scale * kLog2eF, c2 = p.softcap * kLog2eF;
  const int q_last = (qt0 + QT < p.t ? qt0 + QT : p.t) - 1;
  const long q_first = p.cache_position[0];
  const KeyRange kr = key_range(p, b, q_first + qt0, q_first + q_last);
  const int n_keys = kr.n;
  const long kp = (long)p.kv_heads * p.dim, vp = (long)p.kv_heads * p.vdim;
  const uint16_t* kc = (const uint16_t*)p.k_cache + b * p.k_batch + (long)kvh * p.dim;
  const uint16_t* vc = (const uint16_t*)p.v_cache + b * p.v_batch + (long)kvh * p.vdim;
  // Wave w delivers rows 8 w .., 8 (w + NW) .., ... of a block (their swizzles agree). Rows past the last key
  // repeat it (masked), columns past a row's end repeat its start (the queries hold zeros there; such values are
  // never stored).
  const int lrow = wave * 8 + (lane >> 3), lc = ((lane & 7) ^ tile_swz(lrow)) * 8;
  auto load_k = [&](int s0, uint16_t* dst) {
#pragma unroll
    for (int u = 0; u < RB; ++u) {
      const int n = s0 + lrow + RSTEP * u;
      const uint16_t* src = kc + kr.slot(n < n_keys ? n : n_keys - 1) * kp;
#pragma unroll
      for (int cg = 0; cg < KG; ++cg)
        load_lds16(src + (cg * 64 + lc < p.dim ? cg * 64 + lc : 0), &dst[(cg * 64 + wave * 8 + RSTEP * u) * 64]);
    }
  };
  auto load_v = [&](int s0) {
#pragma unroll
    for (int u = 0; u < RB; ++u) {
      const int n = s0 + lrow + RSTEP * u;
      const uint16_t* src = vc + kr.slot(n < n_keys ? n : n_keys - 1) * vp;
#pragma unroll
      for (int cg = 0; cg < VG; ++cg)
        load_lds16(src + (cg * 64 + lc < p.vdim ? cg * 64 + lc : 0), &vl[(cg * 64 + wave * 8 + RSTEP * u) * 64]);
    }
  };
  u32x4 q[2][DKC];
#pragma unroll
  for (int qt = 0; qt < 2; ++qt) {
    const int tq = wq + qt * 16 + i16 < p.t ? wq + qt * 16 + i16 : p.t - 1;
    const uint16_t* src = (const uint16_t*)p.q + (((long)b * p.t + tq) * p.heads + h) * p.dim;
#pragma unroll
    for (int c = 0; c < DKC; ++c) {
      const int e = c * 32 + 8 * g;
      const u32x4 v = ld16(src + (e < p.dim ? e : 0));
      q[qt][c] = e < p.dim ? v : u32x4{0u, 0u, 0u, 0u};
    }
  }
  if (n_keys > 0) load_k(0, smem);
  // this wave's queries, counted like the window's keys
  const int wq0 = (int)(q_first + wq - kr.first) - kr.shift, wq1 = wq0 + 31;
  for (int s0 = 0, buf = 0; s0 < n_keys; s0 += 64, buf ^= 1) {
    const uint16_t* kl = smem + buf * KSTAGE;
    const bool more = s0 + 64 < n_keys;
    // (blocks that none of the wave's queries sees are skipped)
    const bool mine = s0 <= wq1 && (p.window <= 0 || s0 + 63 > wq0 - p.window || s0 < p.keep);
    wait_loads<0>();  // this wave's rows of the keys have landed
    __syncthreads();  // ... and everybody's; everybody is done with the values and the other keys
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
      const bool full = s0 + 63 <= wq0 && (p.window <= 0 || s0 > wq1 - p.window || s0 + 63 < p.keep);
#pragma unroll
      for (int qt = 0; qt < 2; ++qt) {
        float mx = -INFINITY;
        if (full) {
#pragma unroll
          for (int kt = 0; kt < 4; ++kt)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              s4[qt][kt][r] = score_log2<CAP>(s4[qt][kt][r], c1, c2);
              mx = fmaxf(mx, s4[qt][kt][r]);
            }
        } else {
          // keys counted from the block's start: the last one seen, the last one in front of the window, the
          // first one that is not kept
          const int last = wq0 + qt * 16 + i16 - s0, before = p.window > 0 ? last - p.window : -1, kept = p.keep - s0;
#pragma unroll
          for (int kt = 0; kt < 4; ++kt)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              const int s = kt * 16 + 4 * g + r;
              const float v = score_log2<CAP>(s4[qt][kt][r], c1, c2);
              s4[qt][kt][r] = s <= last && (s > before || s < kept) ? v : -INFINITY;
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
          const u32x2 a0 = lds_read_tr16(&vl[tile_at<64>(row, col)]), a1 = lds_read_tr16(&vl[tile_at<64>(row + 16, col)]);
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
    const int tq = wq + qt * 16 + i16;
    if (tq >= p.t) continue;
    const long tok = (long)b * p.t + tq;
    uint16_t* dst = (uint16_t*)p.out + (tok * p.heads + h) * p.vdim;
    const uint16_t* gr = (const uint16_t*)p.gate + tok * p.gate_pitch + (long)h * p.vdim;
#pragma unroll
    for (int j = 0; j < DVT; ++j) {
      const int v = 16 * j + 4 * g;  // (vdim and the gate's pitch are multiples of 4)
      if (v >= p.vdim) continue;
      float o[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = acc[qt][j][r] * inv;
      if (p.gate) {
        const u32x2 w = ld8(gr + v);
        o[0] *= sigmoid_f32(T::lo(w.x));
        o[1] *= sigmoid_f32(T::hi(w.x));
        o[2] *= sigmoid_f32(T::lo(w.y));
        o[3] *= sigmoid_f32(T::hi(w.y));
      }
      *(u32x2*)(dst + v) = u32x2{T::pack2(o[0], o[1]), T::pack2(o[2], o[3])};
    }
  }
}

// ---------------------------------------------------------------------------------------
// launchers
// ---------------------------------------------------------------------------------------
template <typename T>
static int launch_hybrid_prepare(hipStream_t s, const HybridAttnParams& p) {
  const void* ptrs[] = {p.proj, p.q_gain, p.k_gain, p.q_out, p.k_cache, p.v_cache};
  bool vec = p.dim % 8 == 0 && p.vdim % 8 == 0 && p.pitch % 8 == 0 && p.k_off % 8 == 0 && p.v_off % 8 == 0 && p.k_batch % 8 == 0 &&
             p.v_batch % 8 == 0;
  for (const void* q : ptrs) vec = vec && aligned16(q);
  const int tokens = p.batch * p.t;
  const dim3 grid(tokens), block(tokens <= MUI_MAX_TOKENS ? 512 : 256);
  const size_t lds = (size_t)(p.dim + 1) / 2 * 8;
  if (vec) return launch_with_lds(hybrid_prepare_kernel<T, true>, grid, block, lds, s, p);
  return launch_with_lds(hybrid_prepare_kernel<T, false>, grid, block, lds, s, p);
}

template <typename T>
static int launch_hybrid_plain(hipStream_t s, const HybridAttnParams& p) {
  if (p.batch * p.t > 65535) return MUI_ERR_UNSUPPORTED;
  return launch_with_lds(hybrid_plain_kernel<T>, dim3(p.heads, p.batch * p.t), dim3(256), ((size_t)p.dim + p.vdim) * 4, s, p);
}

template <typename T, int DKC, int DVT>
static int launch_hybrid_decode_t(hipStream_t s, const HybridAttnParams& p) {
  const int share = p.heads / p.kv_heads, tokens = p.batch * p.t;
  const dim3 grid(p.splits, p.kv_heads * ceil_div(share, 16), tokens), block(256);
  const size_t lds = (size_t)kHdKeys * (DKC * 32 + DVT * 16) * 2;
  const int st = p.softcap > 0.f ? launch_with_lds(hybrid_decode_kernel<T, DKC, DVT, true>, grid, block, lds, s, p)
                                 : launch_with_lds(hybrid_decode_kernel<T, DKC, DVT, false>, grid, block, lds, s, p);
  if (st != MUI_OK || p.splits == 1) return st;
  hipLaunchKernelGGL((hybrid_combine_kernel<T>), dim3(p.heads, tokens), dim3(128), 0, s, p);
  return launch_status();
}

template <typename T, int DKC, int DVT>
static int launch_hybrid_prefill_t(hipStream_t s, const HybridAttnParams& p0) {
  HybridAttnParams p = p0;
  const int share = p.heads / p.kv_heads;
  auto launch = [&](auto capped, auto plain, int nw, int hw) {
    p.head_waves = hw;
    const int tiles = ceil_div(p.t, 32 * (nw / hw));
    if (tiles > 65535) return (int)MUI_ERR_UNSUPPORTED;
    const dim3 grid(p.batch * (p.heads / hw), tiles), block(64 * nw);
    return p.softcap > 0.f ? launch_with_lds(capped, grid, block, hybrid_prefill_lds<DKC, DVT>(), s, p)
                           : launch_with_lds(plain, grid, block, hybrid_prefill_lds<DKC, DVT>(), s, p);
  };
  // short prompts: half as many queries per workgroup, so that there are workgroups for every CU
  const int hw4 = share % 4 == 0 ? 4 : (share % 2 == 0 ? 2 : 1);
  if (p.batch * (p.heads / hw4) * ceil_div(p.t, 32 * (4 / hw4)) <= device_cus())
    return launch(hybrid_prefill_kernel<T, DKC, DVT, 2, true>, hybrid_prefill_kernel<T, DKC, DVT, 2, false>, 2, share % 2 == 0 ? 2 : 1);
  return launch(hybrid_prefill_kernel<T, DKC, DVT, 4, true>, hybrid_prefill_kernel<T, DKC, DVT, 4, false>, 4, hw4);
}

// keys per split and number of splits of the decode kernel for up to `span` visible keys
static void hybrid_split(int batch, int t, int heads, int kv_heads, int span, int* splits, int* split_keys) {
  const int groups = batch * t * kv_heads * ceil_div(heads / kv_heads, 16);
  int want = device_cus() * 2 / (groups > 0 ? groups : 1);
  want = want < 1 ? 1 : (want > kHdMaxSplits ? kHdMaxSplits : want);
  const int blocks = ceil_div(span, kHdKeys), per = ceil_div(blocks, want);
  *split_keys = per * kHdKeys;
  *splits = ceil_div(blocks, per);
}

template <typename T>
static int launch_hybrid_attention(hipStream_t s, int route, const HybridAttnParams& p) {
  const bool d64 = p.dim <= 64 && p.vdim <= 64, d128 = p.dim <= 128 && p.vdim <= 128;
  if (route == MUI_HYBRID_DECODE)
    return d64 ? launch_hybrid_decode_t<T, 2, 4>(s, p) : (d128 ? launch_hybrid_decode_t<T, 4, 8>(s, p) : launch_hybrid_decode_t<T, 8, 16>(s, p));
  return d64 ? launch_hybrid_prefill_t<T, 2, 4>(s, p) : (d128 ? launch_hybrid_prefill_t<T, 4, 8>(s, p) : launch_hybrid_prefill_t<T, 8, 16>(s, p));
}

}  // namespace mui

using namespace mui;

extern "C" int mui_hybrid_prepare(mui_stream_t stream, int dtype, const void* proj, long pitch, long k_offset, long v_offset,
                                  const void* q_gain, const void* k_gain, float epsilon, const double* inv_freq, int rot_dims,
                                  const int64_t* cache_position, const int64_t* row_start, void* q_out, void* k_cache,
                                  long k_batch_stride, void* v_cache, long v_batch_stride, int batch, int t, int heads,
                                  int kv_heads, int dim, int vdim, int max_cache_len) {
  MUI_CHECK_ARG(proj && cache_position && q_out && k_cache && v_cache && batch > 0 && t > 0 && heads > 0 && kv_heads > 0);
  MUI_CHECK_ARG(heads % kv_heads == 0 && dim > 0 && vdim > 0 && rot_dims >= 0 && rot_dims <= dim && rot_dims % 2 == 0);
  MUI_CHECK_ARG((rot_dims == 0 || inv_freq) && max_cache_len > 0 && (long)batch * t < (1L << 31));
  MUI_CHECK_ARG(k_offset >= 0 && v_offset >= 0 && pitch >= (long)heads * dim && pitch >= k_offset + (long)kv_heads * dim &&
                pitch >= v_offset + (long)kv_heads * vdim);
  HybridAttnParams p = {};
  p.proj = proj; p.pitch = pitch; p.k_off = k_offset; p.v_off = v_offset; p.q_gain = q_gain; p.k_gain = k_gain; p.eps = epsilon;
  p.inv_freq = inv_freq; p.rot = rot_dims; p.cache_position = cache_position; p.row_start = row_start; p.q_out = q_out;
  p.k_cache = k_cache; p.k_batch = k_batch_stride; p.v_cache = v_cache; p.v_batch = v_batch_stride; p.batch = batch; p.t = t;
  p.heads = heads; p.kv_heads = kv_heads; p.dim = dim; p.vdim = vdim; p.max_cache_len = max_cache_len;
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MUI_DTYPE_F16) return launch_hybrid_prepare<F16>(s, p);
  if (dtype == MUI_DTYPE_BF16) return launch_hybrid_prepare<BF16>(s, p);
  if (dtype == MUI_DTYPE_F32) return launch_hybrid_prepare<F32>(s, p);
  return MUI_ERR_INVALID_ARG;
}

extern "C" int mui_hybrid_attention_route(int dtype, int tokens, int dim, int vdim) {
  if (dtype == MUI_DTYPE_F32 || dim % 8 || vdim % 8 || dim > 256 || vdim > 256) return MUI_HYBRID_PLAIN;
  return tokens > MUI_MAX_TOKENS ? MUI_HYBRID_PREFILL : MUI_HYBRID_DECODE;
}

extern "C" size_t mui_hybrid_decode_scratch_bytes(int batch, int t, int heads, int kv_heads, int vdim, int span) {
  if (batch < 1 || t < 1 || heads < 1 || kv_heads < 1 || vdim < 1 || span < 1) return 0;
  int splits, keys;
  hybrid_split(batch, t, heads, kv_heads, span, &splits, &keys);
  return splits == 1 ? 0 : (size_t)batch * t * heads * splits * (vdim + 2) * 4;
}

extern "C" int mui_hybrid_attention(mui_stream_t stream, int dtype, int route, const void* q, const void* k_cache,
                                    long k_batch_stride, const void* v_cache, long v_batch_stride, const void* gate,
                                    long gate_pitch, const int64_t* cache_position, const int64_t* row_start, float scale,
                                    float softcap, int window, int keep_first, void* scratch, int span, void* out, int batch,
                                    int t, int heads, int kv_heads, int dim, int vdim, int max_cache_len) {
  MUI_CHECK_ARG(q && k_cache && v_cache && cache_position && out && batch > 0 && t > 0 && heads > 0 && kv_heads > 0);
  MUI_CHECK_ARG(heads % kv_heads == 0 && dim > 0 && vdim > 0 && max_cache_len > 0 && keep_first >= 0 && window >= 0);
  MUI_CHECK_ARG(!gate || gate_pitch >= (long)heads * vdim);
  HybridAttnParams p = {};
  p.q = q; p.k_cache = (void*)k_cache; p.k_batch = k_batch_stride; p.v_cache = (void*)v_cache; p.v_batch = v_batch_stride;
  p.gate = gate; p.gate_pitch = gate_pitch; p.cache_position = cache_position; p.row_start = row_start; p.scale = scale;
  p.softcap = softcap; p.window = window; p.keep = keep_first; p.out = out; p.batch = batch; p.t = t; p.heads = heads;
  p.kv_heads = kv_heads; p.dim = dim; p.vdim = vdim; p.max_cache_len = max_cache_len;
  hipStream_t s = (hipStream_t)stream;
  if (route == MUI_HYBRID_PLAIN) {
    if (dtype == MUI_DTYPE_F16) return launch_hybrid_plain<F16>(s, p);
    if (dtype == MUI_DTYPE_BF16) return launch_hybrid_plain<BF16>(s, p);
    if (dtype == MUI_DTYPE_F32) return launch_hybrid_plain<F32>(s, p);
    return MUI_ERR_INVALID_ARG;
  }
  MUI_CHECK_ARG(route == MUI_HYBRID_DECODE || route == MUI_HYBRID_PREFILL);
  if (mui_hybrid_attention_route(dtype, MUI_MAX_TOKENS + 1, dim, vdim) != MUI_HYBRID_PREFILL) return MUI_ERR_UNSUPPORTED;
  if (!aligned16(q) || !aligned16(k_cache) || !aligned16(v_cache) || !aligned16(out) || k_batch_stride % 8 || v_batch_stride % 8 ||
      (gate && (((uintptr_t)gate & 7) || gate_pitch % 4)))
    return MUI_ERR_ALIGNMENT;
  if (route == MUI_HYBRID_DECODE) {
    MUI_CHECK_ARG(span > 0);
    if ((long)batch * t > 65535) return MUI_ERR_UNSUPPORTED;
    hybrid_split(batch, t, heads, kv_heads, span, &p.splits, &p.split_keys);
    MUI_CHECK_ARG(p.splits == 1 || scratch);
    if ((uintptr_t)scratch & 15) return MUI_ERR_ALIGNMENT;
    p.part = (float*)scratch;
    p.part_ml = p.part + (size_t)batch * t * heads * p.splits * vdim;
  }
  if (dtype == MUI_DTYPE_F16) return launch_hybrid_attention<F16>(s, route, p);
  return launch_hybrid_attention<BF16>(s, route, p);
}
