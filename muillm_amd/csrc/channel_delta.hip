// Gated delta rule with one decay per head and key channel, per head:
//   S <- g_t * S (rows), u_t = beta_t (v_t - S^T k_t), S <- S + k_t u_t^T, o_t = S^T q_t
// q, k, v come from a projection through a short causal convolution per channel and silu; q and k are unit vectors
// per (query / key) head, q scaled by q_scale; beta = sigmoid(b); g = exp(-exp(A_log) softplus(A2 a + dt_bias)), a a
// low-rank projection; the result is normed per head, times a gain, times sigmoid(G2 g) of another one.
// S and everything that enters it stays in fp32; only the projections arrive in the activations' type.
//
//   step    (few tokens) one workgroup per head and batch row does all of it, S in registers.
//   chunks  (prompts) 64 tokens at a time, in sub-chunks of 16. With G_t the product of the decays of a chunk up to t,
//             A_ts = sum_d k_t k_s (G_t / G_s),  (1 + diag(beta) A) U = diag(beta) (V - (G * K) S_in)   (A strictly lower)
//             O = (G * Q) S_in + A^qk U,  S_out = G_end * S_in + ((G_end / G) * K)^T U
//           No quotient is ever formed: rows are multiplied by the decays since the start of their sub-chunk,
//           columns by the decays up to the end of theirs, whole sub-chunks in between are a factor of their own,
//           and pairs inside a sub-chunk carry a running product. Strong decays underflow to the zero they mean.
//           1. prepare: convolutions, norms, decays, A, and W, U0 from U = U0 - W S_in, all chunks at once
//           2. scan: one workgroup per head and 16 value columns walks the chunks, S in accumulators
//           3. output: norm, gain, gate; the last inputs of the convolutions for the next call
//           All products with S or U are v_mfma_f32_16x16x4_f32.
// The last taps - 1 inputs of the convolutions are kept in a ring of rows by slot. Tokens in front of a row's
// first slot (left padding) leave the state alone and are zeros to the convolutions.
#include "hybrid.cuh"

namespace mui {

constexpr int kDChunk = 64, kDSub = 16;
constexpr float kUnitEps = 1e-6f;

struct DeltaParams {
  const void* proj;  // [tokens, pitch]; q | k | v | a | g | b at the offsets below
  long pitch;
  int q_off, k_off, v_off, a_off, g_off, b_off;
  const void* conv;  // [channels, taps], channels q | k | v
  const void* a2;    // [heads * dk, ra]
  const void* dt_bias;  // [heads * dk]
  const void* a_log;    // [heads]
  const void* g2;    // [heads * dv, rg]
  const void* gain;  // [dv]
  float q_scale, eps;
  float* s;          // [batch, heads, dk, dv]
  void* ring;        // [batch, ring_rows, channels]
  const int64_t* cache_position;  // [t], consecutive slots
  const int64_t* row_start;       // [batch] or null
  void* y;           // [tokens, heads * dv]
  int batch, t, heads, kv_heads, dk, dv, ra, rg, taps, ring_rows, channels;
  bool vec;  // the low-rank operands may be read 16 bytes at a time (where their rank is a multiple of 8)
  // chunks
  float *qe, *w, *kd, *gc, *aqk, *u0, *o;  // per (batch, head, chunk); o [tokens, heads, dv]
  int chunks, dkp, dvp;
};

// Each is a few fp32 operations around the hardware's exp2, log2 and reciprocal (1 ulp).
constexpr float kLog2E = 1.4426950408889634f;
__device__ __forceinline__ float sigm(float z) { return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-kLog2E * z)); }
__device__ __forceinline__ float silu(float z) { return z * sigm(z); }
// exp(neg_a softplus(z)), softplus(z) = max(z, 0) + log(1 + u), u = exp(-|z|); the logarithm of w = 1 + u is scaled by
// u / (w - 1), which makes good what the sum lost
__device__ __forceinline__ float decay_of(float neg_a, float z) {
  const float u = __builtin_amdgcn_exp2f(-kLog2E * fabsf(z)), w = 1.f + u, d = w - 1.f;
  const float l = d > 0.f ? __builtin_amdgcn_logf(w) * (u * __builtin_amdgcn_rcpf(d)) : u * kLog2E;
  return __builtin_amdgcn_exp2f(neg_a * fmaf(fmaxf(z, 0.f), kLog2E, l));
}

template <typename T>
struct DeltaRow {  // one batch row
  typedef typename T::storage S;
  const S* proj;
  const S* ring;
  long p0, start;  // slot of token 0, first slot of the row
  int ring0;       // ring row of token 0
  __device__ __forceinline__ DeltaRow(const DeltaParams& p, int b)
      : proj((const S*)p.proj + (long)b * p.t * p.pitch), ring((const S*)p.ring + (long)b * p.ring_rows * p.channels),
        p0(p.cache_position[0]), start(p.row_start ? p.row_start[b] : 0), ring0((int)((uint32_t)p0 % (uint32_t)p.ring_rows)) {}
  // ring row of token tok, -ring_rows <= tok < 0
  __device__ __forceinline__ int ring_row(const DeltaParams& p, int tok) const { return ring0 + tok + (ring0 + tok < 0 ? p.ring_rows : 0); }
  __device__ __forceinline__ bool live(int tok) const { return p0 + tok >= start; }
  // input of channel c (column `col` of the projection) at token tok, which may lie in front of this call
  __device__ __forceinline__ float raw(const DeltaParams& p, int tok, int col, int c) const {
    const long slot = p0 + tok;
    if (slot < start || slot < 0) return 0.f;
    return T::one(tok >= 0 ? proj[(long)tok * p.pitch + col] : ring[(long)ring_row(p, tok) * p.channels + c]);
  }
  // convolution and silu
  __device__ __forceinline__ float conv(const DeltaParams& p, int tok, int col, int c) const {
    const S* w = (const S*)p.conv + (long)c * p.taps;
    float a = 0.f;
    for (int j = p.taps - 1; j >= 0; --j) a = fmaf(T::one(w[p.taps - 1 - j]), raw(p, tok - j, col, c), a);
    return silu(a);
  }
  // the same for up to four taps, all operands requested at once (taps that are not there, or inputs in front of the
  // sequence, read something valid and count as zero)
  __device__ __forceinline__ float conv4(const DeltaParams& p, int tok, int col, int c) const {
    const S* w = (const S*)p.conv + (long)c * p.taps;
    float x[4], a = 0.f;
    S f[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const S* src = tok >= j ? proj + (long)(tok - j) * p.pitch + col : ring + (long)ring_row(p, tok - j) * p.channels + c;
      x[j] = T::one(*src);
      f[j] = w[j < p.taps ? p.taps - 1 - j : 0];
    }
#pragma unroll
    for (int j = 3; j >= 0; --j) {
      const bool on = j < p.taps && p0 + tok - j >= (start > 0 ? start : 0);
      a = on ? fmaf(T::one(f[j]), x[j], a) : a;
    }
    return silu(a);
  }
};

// the last taps - 1 inputs of the call into the ring; head h writes its value channels, the first head of a group
// its query and key channels
template <typename T>
__device__ __forceinline__ void keep_inputs(const DeltaParams& p, int b, int h, int t, int nt) {
  typedef typename T::storage S;
  const int share = p.heads / p.kv_heads, kvh = h / share, nq = p.kv_heads * p.dk;
  const bool first = h % share == 0;
  const int from = p.t - (p.taps - 1) > 0 ? p.t - (p.taps - 1) : 0;
  const int per = (first ? 2 * p.dk : 0) + p.dv;
  const long p0 = p.cache_position[0];
  S* ring = (S*)p.ring + (long)b * p.ring_rows * p.channels;
  for (int i = t; i < per * (p.t - from); i += nt) {
    const int tok = from + i / per;
    int e = i % per, c, col;
    if (e < p.dv) {
      c = 2 * nq + h * p.dv + e;
      col = p.v_off + h * p.dv + e;
    } else {
      e -= p.dv;
      const int k = e >= p.dk;
      c = k * nq + kvh * p.dk + (e - k * p.dk);
      col = (k ? p.k_off : p.q_off) + kvh * p.dk + (e - k * p.dk);
    }
    ring[(long)((uint32_t)(p0 + tok) % (uint32_t)p.ring_rows) * p.channels + c] = ((const S*)p.proj)[((long)b * p.t + tok) * p.pitch + col];
  }
}

// ---------------------------------------------------------------------------------------
// step: grid (heads, batch), 512 threads; thread = (four columns, rows rg, rg + RG, ..)
// ---------------------------------------------------------------------------------------
extern __shared__ __align__(16) unsigned char cd_smem[];
constexpr int kStepThreads = 512;

// out[row] = f(sum_k W[row, k] x[k]) for rows of a low-rank second factor; eight threads per row, x in LDS
template <typename T, typename F>
__device__ __forceinline__ void low_rank_rows(const typename T::storage* w, const float* x, int rows, int r, bool vec, F f) {
  const int t = threadIdx.x, sub = t & 7;
  for (int row0 = 0; row0 < rows; row0 += kStepThreads / 8) {
    const int row = row0 + (t >> 3);
    const typename T::storage* wr = w + (long)(row < rows ? row : rows - 1) * r;
    float a = 0.f;
    if (vec) {
#pragma unroll 2
      for (int c = sub * 8; c < r; c += 64) {
        float fw[8];
        load8<T>(wr + c, fw);
#pragma unroll
        for (int i = 0; i < 8; ++i) a = fmaf(fw[i], x[c + i], a);
      }
    } else {
      for (int c = sub; c < r; c += 8) a = fmaf(T::one(wr[c]), x[c], a);
    }
    a += dpp_f32<kDppXor1>(a);
    a += dpp_f32<kDppXor2>(a);
    a += dpp_f32<kDppHalfMirror>(a);
    if (sub == 0 && row < rows) f(row, a);
  }
}

// The same with the matrix in registers: up to kLowRankHeld vectors of 8 per thread (16-bit types), requested before x is known.
constexpr int kLowRankHeld = 4;
template <typename T>
struct LowRankHeld {
  u32x4 w[kLowRankHeld];
  int rows, iters;  // iters: vectors of a row per thread
  __device__ __forceinline__ void load(int t, const typename T::storage* m, int n, int r) {
    const int sub = t & 7;
    rows = n;
    iters = (r + 63) / 64;
    int row = t >> 3, c = sub * 8;
#pragma unroll
    for (int i = 0; i < kLowRankHeld; ++i) {
      w[i] = ld16(m + (row < n ? row : n - 1) * r + (c < r ? c : 0));
      if (c >= r) w[i] = u32x4{0u, 0u, 0u, 0u};
      step(t, row, c);
    }
  }
  template <typename F>
  __device__ __forceinline__ void run(int t, const float* x, int r, F f) const {
    const int sub = t & 7;
    float a = 0.f;
    int row = t >> 3, c = sub * 8;
#pragma unroll
    for (int i = 0; i < kLowRankHeld; ++i) {
      const float* xc = x + (c < r ? c : 0);
#pragma unroll
      for (int j = 0; j < 4; ++j) a = fmaf(T::hi(w[i][j]), xc[2 * j + 1], fmaf(T::lo(w[i][j]), xc[2 * j], a));
      const int at = row;
      if (step(t, row, c)) {  // uniform for the workgroup
        a += dpp_f32<kDppXor1>(a);
        a += dpp_f32<kDppXor2>(a);
        a += dpp_f32<kDppHalfMirror>(a);
        if (sub == 0 && at < rows) f(at, a);
        a = 0.f;
      }
    }
  }
  // the next vector; true at the end of a row
  __device__ __forceinline__ bool step(int t, int& row, int& c) const {
    c += 64;
    if (c < iters * 64) return false;
    c = (t & 7) * 8;
    row += 64;
    return true;
  }
};

// NR > 0: NR rows of S per thread in registers, for the sizes that delta_step_held names. 0: every size, S stays in memory.
template <typename T, int NR>
__global__ void __launch_bounds__(kStepThreads) delta_step_kernel(const DeltaParams p, int cgp) {
  typedef typename T::storage S;
  __shared__ float red[8][4];
  int t = threadIdx.x;
  const int lane = t & 63, wave = t >> 6;
  const int h = blockIdx.x, b = blockIdx.y, share = p.heads / p.kv_heads, kvh = h / share, nq = p.kv_heads * p.dk;
  const int parts = cgp <= 64 ? 8 : kStepThreads / cgp, cols = 4 * cgp;
  // rows and columns past a head's end are zeros
  const int dkp = NR > 0 ? NR * (kStepThreads / cgp) : p.dk;
  float* qs = (float*)cd_smem;  // dkp
  float* ks = qs + dkp;         // dkp
  float* gs = ks + dkp;         // dkp: first the decays' biases, then the decays
  float* vs = gs + dkp;         // cols; later u
  float* og = vs + cols;        // dv: gain, then gain times output gate
  float* gz = og + p.dv;        // dv: output gate before its sigmoid
  float* av = gz + p.dv;        // ra
  float* gv = av + p.ra;        // rg
  float* part = gv + p.rg + ((4 - ((3 * dkp + 2 * p.dv + p.ra + p.rg) & 3)) & 3);  // [2][parts][cols]
  const DeltaRow<T> row(p, b);
  const int cg = t & (cgp - 1), rg = t / cgp, RG = kStepThreads / cgp, c0 = cg * 4;
  float* st = p.s + ((long)b * p.heads + h) * p.dk * p.dv;
  const float neg_a = -expf(T::one(((const S*)p.a_log)[h]));
  f32x4 sreg[NR > 0 ? NR : 1];
  auto load_s = [&](int d) {
    f32x4 x = {0.f, 0.f, 0.f, 0.f};
    const bool in = d < p.dk && c0 < p.dv;
    if constexpr (NR > 0) {  // dv is a multiple of 4
      const f32x4 y = *(const f32x4*)(st + (in ? d * p.dv + c0 : 0));
#pragma unroll
      for (int j = 0; j < 4; ++j) x[j] = in ? y[j] : 0.f;
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (in && c0 + j < p.dv) x[j] = st[d * p.dv + c0 + j];
    }
    return x;
  };
  auto store_s = [&](int d, f32x4 x) {
    if (d >= p.dk || c0 >= p.dv) return;
    if constexpr (NR > 0) {
      *(f32x4*)(st + d * p.dv + c0) = x;
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (c0 + j < p.dv) st[d * p.dv + c0 + j] = x[j];
    }
  };
  const S *a2 = (const S*)p.a2 + (long)h * p.dk * p.ra, *g2 = (const S*)p.g2 + (long)h * p.dv * p.rg;
  LowRankHeld<T> held_a, held_g;
  if constexpr (NR > 0) {
    held_a.load(t, a2, p.dk, p.ra);
    held_g.load(t, g2, p.dv, p.rg);
#pragma unroll
    for (int i = 0; i < NR; ++i) sreg[i] = load_s(rg + RG * i);
  }
  auto conv = [&](int tok, int col, int c) {
    if constexpr (NR > 0) return row.conv4(p, tok, col, c);
    else return row.conv(p, tok, col, c);
  };
  for (int i = p.dk + t; i < dkp; i += kStepThreads) qs[i] = ks[i] = gs[i] = 0.f;
  for (int i = p.dv + t; i < cols; i += kStepThreads) vs[i] = 0.f;
  for (int tok = 0; tok < p.t; ++tok) {
    asm volatile("" : "+v"(t));  // (one token is the rule: addresses kept from token to token would only cost registers)
    S* yrow = (S*)p.y + (((long)b * p.t + tok) * p.heads + h) * p.dv;
    if (!row.live(tok)) {  // uniform for the workgroup
      for (int i = t; i < p.dv; i += kStepThreads) yrow[i] = T::pack(0.f);
      continue;
    }
    const S* pr = row.proj + (long)tok * p.pitch;
    // inputs of the recurrence
    float qq = 0.f, kk = 0.f, qk = 0.f;
    for (int d = t; d < p.dk; d += kStepThreads) {
      const int c = kvh * p.dk + d;
      const float x = conv(tok, p.q_off + c, c), y = conv(tok, p.k_off + c, nq + c);
      qs[d] = x;
      ks[d] = y;
      gs[d] = T::one(((const S*)p.dt_bias)[h * p.dk + d]);
      qq = fmaf(x, x, qq);
      kk = fmaf(y, y, kk);
      qk = fmaf(x, y, qk);
    }
    for (int e = kStepThreads - 1 - t; e < p.dv; e += kStepThreads) {  // (from the other end: dk threads are busy above)
      const int c = h * p.dv + e;
      vs[e] = conv(tok, p.v_off + c, 2 * nq + c);
      og[e] = T::one(((const S*)p.gain)[e]);
    }
    for (int i = t; i < p.ra; i += kStepThreads) av[i] = T::one(pr[p.a_off + i]);
    for (int i = kStepThreads - 1 - t; i < p.rg; i += kStepThreads) gv[i] = T::one(pr[p.g_off + i]);
    const float beta = sigm(T::one(pr[p.b_off + h]));
    qq = wave_sum(qq);
    kk = wave_sum(kk);
    qk = wave_sum(qk);
    if (lane == 0) {
      red[wave][0] = qq;
      red[wave][1] = kk;
      red[wave][2] = qk;
    }
    __syncthreads();
    auto decay = [&](int d, float z) { gs[d] += z; };
    auto open = [&](int e, float z) { gz[e] = z; };
    if constexpr (NR > 0) {
      held_a.run(t, av, p.ra, decay);
      held_g.run(t, gv, p.rg, open);
    } else {
      low_rank_rows<T>(a2, av, p.dk, p.ra, p.ra % 8 == 0 && p.vec, decay);
      low_rank_rows<T>(g2, gv, p.dv, p.rg, p.rg % 8 == 0 && p.vec, open);
    }
    qq = kk = qk = 0.f;
#pragma unroll
    for (int w = 0; w < 8; ++w) {
      qq += red[w][0];
      kk += red[w][1];
      qk += red[w][2];
    }
    const float rq = p.q_scale / sqrtf(qq + kUnitEps), rk = 1.f / sqrtf(kk + kUnitEps);
    __syncthreads();
    for (int d = t; d < p.dk; d += kStepThreads) gs[d] = decay_of(neg_a, gs[d]);
    for (int e = kStepThreads - 1 - t; e < p.dv; e += kStepThreads) og[e] *= sigm(gz[e]);
    __syncthreads();
    // decayed S against k and q
    f32x4 pk = {0.f, 0.f, 0.f, 0.f}, pq = pk;
    auto sweep = [&](f32x4& x, int d) {
      const float g = gs[d], k = ks[d] * rk, q = qs[d] * rq;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        x[j] *= g;
        pk[j] = fmaf(x[j], k, pk[j]);
        pq[j] = fmaf(x[j], q, pq[j]);
      }
    };
    if constexpr (NR > 0) {
#pragma unroll
      for (int i = 0; i < NR; ++i) {
        sweep(sreg[i], rg + RG * i);
        if (i % 4 == 3) asm volatile("" ::: "memory");  // (LDS reads of four rows ahead are enough)
      }
    } else {
      for (int d = rg; d < p.dk; d += RG) {
        f32x4 x = load_s(d);
        sweep(x, d);
      }
    }
    for (int o = cgp; o < 64; o <<= 1)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        pk[j] += __shfl_xor(pk[j], o);
        pq[j] += __shfl_xor(pq[j], o);
      }
    if (lane < cgp) {
      const int pi = cgp <= 64 ? wave : rg;
      *(f32x4*)&part[pi * cols + c0] = pk;
      *(f32x4*)&part[(parts + pi) * cols + c0] = pq;
    }
    __syncthreads();
    const float dot = qk * rq * rk;
    float ss = 0.f;
    for (int e = t; e < p.dv; e += kStepThreads) {
      float a = 0.f, o = 0.f;
      for (int i = 0; i < parts; ++i) {
        a += part[i * cols + e];
        o += part[(parts + i) * cols + e];
      }
      const float u = beta * (vs[e] - a);
      o = fmaf(dot, u, o);
      vs[e] = u;
      part[e] = o;  // (this thread's column of the sums just read)
      ss = fmaf(o, o, ss);
    }
    ss = wave_sum(ss);
    if (lane == 0) red[wave][3] = ss;
    __syncthreads();
    const f32x4 u = {vs[c0], vs[c0 + 1], vs[c0 + 2], vs[c0 + 3]};
    auto write = [&](f32x4& x, int d) {
      const float k = ks[d] * rk;
#pragma unroll
      for (int j = 0; j < 4; ++j) x[j] = fmaf(k, u[j], x[j]);
    };
    if constexpr (NR > 0) {
#pragma unroll
      for (int i = 0; i < NR; ++i) {
        write(sreg[i], rg + RG * i);
        if (i % 4 == 3) asm volatile("" ::: "memory");
      }
    } else {
      for (int d = rg; d < p.dk; d += RG) {
        f32x4 x = load_s(d);
#pragma unroll
        for (int j = 0; j < 4; ++j) x[j] *= gs[d];
        write(x, d);
        store_s(d, x);
      }
    }
    ss = 0.f;
#pragma unroll
    for (int w = 0; w < 8; ++w) ss += red[w][3];
    const float rs = 1.f / sqrtf(ss / (float)p.dv + p.eps);
    for (int e = t; e < p.dv; e += kStepThreads) yrow[e] = T::pack(part[e] * rs * og[e]);
    __syncthreads();  // everything in LDS is free
  }
  if constexpr (NR > 0) {
#pragma unroll
    for (int i = 0; i < NR; ++i) store_s(rg + RG * i, sreg[i]);
  }
  keep_inputs<T>(p, b, h, t, kStepThreads);
}

// ---------------------------------------------------------------------------------------
// chunks
// ---------------------------------------------------------------------------------------
// N 16 x 16 tiles of X W^T over r: lane's row of X and of each tile's W (row lane % 16 each); D: column W row lane % 16,
// rows X 4 (lane / 16) + r
template <typename T, int N>
__device__ __forceinline__ void low_rank_tiles(const typename T::storage* x, const typename T::storage* const (&w)[N], int r, bool vec, f32x4 (&acc)[N]) {
  const int g = (threadIdx.x & 63) >> 4;
#pragma unroll
  for (int n = 0; n < N; ++n) acc[n] = f32x4{0.f, 0.f, 0.f, 0.f};
  if constexpr (T::kDtype == MUI_DTYPE_F32) {
    for (int k = 0; k < r; k += 4) {
      const int e = k + g < r ? k + g : 0;
      const float a = k + g < r ? x[e] : 0.f;
#pragma unroll
      for (int n = 0; n < N; ++n) acc[n] = mfma_f32(a, w[n][e], acc[n]);
    }
  } else if (vec) {
    for (int k = 0; k < r; k += 128) {
      u32x4 a[4], b[4][N];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int e = k + 32 * u + 8 * g, c = e < r ? e : 0;
        a[u] = ld16(x + c);
        if (e >= r) a[u] = u32x4{0u, 0u, 0u, 0u};
#pragma unroll
        for (int n = 0; n < N; ++n) b[u][n] = ld16(w[n] + c);
      }
#pragma unroll
      for (int u = 0; u < 4; ++u)
#pragma unroll
        for (int n = 0; n < N; ++n) acc[n] = mfma16x16x32<T>(a[u], b[u][n], acc[n]);
    }
  } else {
#pragma unroll 1
    for (int k = 0; k < r; k += 32) {
      const int e = k + 8 * g;
      auto words = [&](const typename T::storage* m) {
        u32x4 v;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int e0 = e + 2 * i, e1 = e0 + 1;
          v[i] = (e0 < r ? (uint32_t)m[e0] : 0u) | ((e1 < r ? (uint32_t)m[e1] : 0u) << 16);
        }
        return v;
      };
      const u32x4 a = words(x);
#pragma unroll
      for (int n = 0; n < N; ++n) acc[n] = mfma16x16x32<T>(a, words(w[n]), acc[n]);
    }
  }
}

// 16 consecutive tokens of a convolved channel, from token tok0 >= 0 (uniform for the wave); TAPS >= p.taps: older ones
// weigh zero. Tokens behind the call read its last one: nothing that reaches a result depends on them (beta is zero there).
template <typename T, int TAPS>
struct ConvRun {
  typedef typename T::storage S;
  S w[TAPS], x[TAPS + 15];
  // column `col` of the projection and channel `c` of lane 0's channel, `lane`: this one's offset
  __device__ __forceinline__ void load(const DeltaParams& p, const DeltaRow<T>& row, int tok0, int col, int c, int lane) {
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
      const int i = j - (TAPS - p.taps);
      w[j] = ((const S*)p.conv)[(long)(c + lane) * p.taps + (i > 0 ? i : 0)];
    }
#pragma unroll
    for (int j = 0; j < TAPS + 15; ++j) {
      const int tok = tok0 - (TAPS - 1) + j;
      const S* src = tok >= 0 ? row.proj + (tok < p.t ? tok : p.t - 1) * p.pitch + col : row.ring + (long)row.ring_row(p, tok) * p.channels + c;
      x[j] = src[lane];
    }
  }
  // lead: the first token whose input counts (delta_lead)
  __device__ __forceinline__ void run(const DeltaParams& p, int tok0, int lead, float (&y)[16]) const {
    float f[TAPS], z[TAPS + 15];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) f[j] = j >= TAPS - p.taps ? T::one(w[j]) : 0.f;
#pragma unroll
    for (int j = 0; j < TAPS + 15; ++j) z[j] = T::one(x[j]);
    if (tok0 - (TAPS - 1) < lead) {
      int first = lead - (tok0 - (TAPS - 1));
      asm volatile("" : "+v"(first));  // (compared in vector registers: so many scalar conditions would spill)
#pragma unroll
      for (int j = 0; j < TAPS + 15; ++j) z[j] = j >= first ? z[j] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float a = 0.f;
#pragma unroll
      for (int j = 0; j < TAPS; ++j) a = fmaf(f[j], z[i + j], a);
      y[i] = silu(a);
    }
  }
};

// the first token (from this call's start; negative: in the ring) that a convolution may see
template <typename T>
__device__ __forceinline__ int delta_lead(const DeltaParams& p, const DeltaRow<T>& row) {
  const long lead = (row.start > 0 ? row.start : 0) - row.p0;
  return lead < 1 - p.taps ? 1 - p.taps : (lead < p.t ? (int)lead : p.t);
}

// 1. grid (chunks, heads, batch); wave w owns sub-chunk w, lane = channel of a block of 64 (NB blocks: dk <= 64 NB)
constexpr int kDPitch = 68;  // 16 rows x 4 consecutive k in 64 different banks
constexpr int kDInvPitch = 20;
template <typename T, int NB, int TAPS>
__global__ void __launch_bounds__(256, NB > 2 || TAPS > 4 ? 1 : 2) delta_prepare_kernel(const DeltaParams p) {
  typedef typename T::storage S;
  constexpr int DKP = 64 * NB;  // = p.dkp
  float* qh = (float*)cd_smem;              // [64][kDPitch]: q times the decays since the start of its sub-chunk
  float* kh = qh + kDChunk * kDPitch;       // the same of k
  float* ke = kh + kDChunk * kDPitch;       // k times the decays up to the end of its sub-chunk
  float* lm = ke + kDChunk * kDPitch;       // [64][kDPitch]: -beta_t A_ts
  __shared__ float gm[4][64 * NB], bt[kDChunk];
  const int t = threadIdx.x, lane = t & 63, wave = __builtin_amdgcn_readfirstlane(t >> 6), g4 = lane >> 4, i16 = lane & 15;
  const int chunk = blockIdx.x, h = blockIdx.y, b = blockIdx.z, kvh = h / (p.heads / p.kv_heads), nq = p.kv_heads * p.dk;
  const long bhc = ((long)b * p.heads + h) * p.chunks + chunk;
  const DeltaRow<T> row(p, b);
  const int tok0 = chunk * kDChunk + wave * kDSub;  // of this wave
  float* qe_out = p.qe + bhc * kDChunk * DKP;
  float* w_out = p.w + bhc * kDChunk * DKP;
  float* kd_out = p.kd + bhc * kDChunk * DKP;
  float* aqk_out = p.aqk + bhc * kDChunk * kDChunk;

  // q, k and decays of this wave's 16 tokens, channel `lane` of every block
  float q[NB][16], k[NB][16], g[NB][16];
  const int lead = delta_lead<T>(p, row);
  {
    ConvRun<T, TAPS> cq[NB], ck[NB];
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) {
      const int c = kvh * p.dk, d = nb * 64 + lane < p.dk ? nb * 64 + lane : 0;
      cq[nb].load(p, row, tok0, p.q_off + c, c, d);
      ck[nb].load(p, row, tok0, p.k_off + c, nq + c, d);
    }
    asm volatile("" ::: "memory");  // all of it is requested before the first use
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) {
      cq[nb].run(p, tok0, lead, q[nb]);
      ck[nb].run(p, tok0, lead, k[nb]);
      if (nb * 64 + lane >= p.dk) {
#pragma unroll
        for (int i = 0; i < 16; ++i) q[nb][i] = k[nb][i] = 0.f;
      }
    }
  }
  {
    const float neg_a = -expf(T::one(((const S*)p.a_log)[h]));
    const bool vec = p.ra % 8 == 0 && p.vec;
    const int tk = tok0 + i16 < p.t ? tok0 + i16 : p.t - 1;
    const S* x = row.proj + (long)tk * p.pitch + p.a_off;
    float* z = qh + wave * kDSub * kDPitch;  // this wave's rows
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) {
      const S* wr[4];
      float bias[4];
      f32x4 v[4];
#pragma unroll
      for (int ct = 0; ct < 4; ++ct) {
        const int d = nb * 64 + ct * 16 + i16, dc = h * p.dk + (d < p.dk ? d : 0);
        wr[ct] = (const S*)p.a2 + (long)dc * p.ra;
        bias[ct] = T::one(((const S*)p.dt_bias)[dc]);
      }
      low_rank_tiles<T, 4>(x, wr, p.ra, vec, v);
#pragma unroll
      for (int ct = 0; ct < 4; ++ct)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int tr = tok0 + 4 * g4 + r;
          const float e = decay_of(neg_a, v[ct][r] + bias[ct]);
          z[(4 * g4 + r) * kDPitch + ct * 16 + i16] = tr < p.t && row.live(tr) ? e : 1.f;
        }
      __builtin_amdgcn_wave_barrier();
#pragma unroll
      for (int i = 0; i < 16; ++i) g[nb][i] = z[i * kDPitch + lane];
      __builtin_amdgcn_wave_barrier();
    }
  }
  if (t < kDChunk) {
    const int tk = chunk * kDChunk + t;
    bt[t] = tk < p.t && row.live(tk) ? sigm(T::one(row.proj[(long)tk * p.pitch + p.b_off + h])) : 0.f;
  }
  // unit vectors
#pragma unroll
  for (int i = 0; i < 16; ++i) {
    float sq = 0.f, sk = 0.f;
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) {
      sq = fmaf(q[nb][i], q[nb][i], sq);
      sk = fmaf(k[nb][i], k[nb][i], sk);
    }
    const float rq = p.q_scale / sqrtf(wave_sum(sq) + kUnitEps), rk = 1.f / sqrtf(wave_sum(sk) + kUnitEps);
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) {
      q[nb][i] *= rq;
      k[nb][i] *= rk;
    }
  }
#pragma unroll
  for (int nb = 0; nb < NB; ++nb) {
    float a = 1.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) a *= g[nb][i];
    gm[wave][nb * 64 + lane] = a;
  }
  __syncthreads();  // bt, gm
  // pairs inside this wave's sub-chunk: k_s times a running product of decays, against k_t and q_t
#pragma unroll
  for (int s = 0; s < 16; ++s) {
    float w[NB], vk[16], vq[16];
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) w[nb] = k[nb][s];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      vk[i] = vq[i] = 0.f;
      if (i >= s) {
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) {
          if (i > s) {
            w[nb] *= g[nb][i];
            vk[i] = fmaf(w[nb], k[nb][i], vk[i]);
          }
          vq[i] = fmaf(w[nb], q[nb][i], vq[i]);
        }
      }
    }
    row16_reduce_scatter<16>(vk, lane);  // lane i of a row of 16 lanes: token i
    row16_reduce_scatter<16>(vq, lane);
    float a = vk[0], c = vq[0];
    a += __shfl_xor(a, 16);
    c += __shfl_xor(c, 16);
    a += __shfl_xor(a, 32);
    c += __shfl_xor(c, 32);
    if (g4 == 0) {
      const int tr = wave * kDSub + i16, sc = wave * kDSub + s;
      lm[tr * kDPitch + sc] = -a * bt[tr];  // zero on and above the diagonal
      aqk_out[tr * kDChunk + sc] = c;      // zero above it
    }
  }
  // pairs of different sub-chunks (row I, column J < I): (3,0) (3,1) | (3,2) (2,0) | (2,1) | (1,0)
  const int pi[2] = {wave < 2 ? 3 : (wave == 2 ? 2 : 1), wave == 0 ? 3 : 2}, pj[2] = {wave == 1 ? 2 : (wave == 2 ? 1 : 0), wave == 0 ? 1 : 0};
  f32x4 akk[2], aqk[2];
#pragma unroll
  for (int u = 0; u < 2; ++u) akk[u] = aqk[u] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int nb = 0; nb < NB; ++nb) {
    const int d = nb * 64 + lane;
    float before = 1.f, after = 1.f;  // whole sub-chunks in front of and behind this one
    for (int m = 0; m < 4; ++m) {
      if (m < wave) before *= gm[m][d];
      if (m > wave) after *= gm[m][d];
    }
    float kd[16];
    float a = 1.f;
#pragma unroll
    for (int i = 15; i >= 0; --i) {
      const float e = k[nb][i] * a;
      ke[(wave * kDSub + i) * kDPitch + lane] = e;
      kd[i] = e * after;
      a *= g[nb][i];
    }
    a = 1.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      a *= g[nb][i];
      const float x = q[nb][i] * a, y = k[nb][i] * a;
      const int tr = wave * kDSub + i;
      qh[tr * kDPitch + lane] = x;
      kh[tr * kDPitch + lane] = y;
      qe_out[tr * DKP + d] = x * before;
      w_out[tr * DKP + d] = y * before;  // (solved in place below)
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
      *(f32x4*)&kd_out[(long)d * kDChunk + wave * kDSub + 4 * i] = f32x4{kd[4 * i], kd[4 * i + 1], kd[4 * i + 2], kd[4 * i + 3]};
    if (wave == 3) p.gc[bhc * DKP + d] = before * gm[3][d];
    __syncthreads();
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      if (u == 1 && wave > 1) continue;
      const int I = pi[u], J = pj[u];
#pragma unroll 4
      for (int k0 = 0; k0 < 64; k0 += 4) {
        float e = ke[(J * kDSub + i16) * kDPitch + k0 + g4];
        for (int m = J + 1; m < I; ++m) e *= gm[m][nb * 64 + k0 + g4];
        akk[u] = mfma_f32(kh[(I * kDSub + i16) * kDPitch + k0 + g4], e, akk[u]);
        aqk[u] = mfma_f32(qh[(I * kDSub + i16) * kDPitch + k0 + g4], e, aqk[u]);
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    if (u == 1 && wave > 1) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int tr = pi[u] * kDSub + 4 * g4 + r, sc = pj[u] * kDSub + i16;
      lm[tr * kDPitch + sc] = -akk[u][r] * bt[tr];
      aqk_out[tr * kDChunk + sc] = aqk[u][r];
    }
  }
  // the values' inputs in front of their convolution (columns v0 + i16 and v0 + 64 + i16, rows 4 g .. of every sub-chunk)
  S vw[2][TAPS], vx[2][4][TAPS + 3];
  auto load_v = [&](int v0) {
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      const int v = v0 + 64 * n + i16, ch = h * p.dv + (v < p.dv ? v : 0);
#pragma unroll
      for (int j = 0; j < TAPS; ++j) {
        const int i = j - (TAPS - p.taps);
        vw[n][j] = ((const S*)p.conv)[(long)(2 * nq + ch) * p.taps + (i > 0 ? i : 0)];
      }
#pragma unroll
      for (int I = 0; I < 4; ++I)
#pragma unroll
        for (int j = 0; j < TAPS + 3; ++j) {
          const int tok = chunk * kDChunk + I * kDSub + 4 * g4 - (TAPS - 1) + j;
          const S* src = row.proj + (tok < 0 ? 0 : (tok < p.t ? tok : p.t - 1)) * p.pitch + p.v_off + ch;
          if (chunk == 0 && I == 0 && tok < 0) src = row.ring + (long)row.ring_row(p, tok) * p.channels + 2 * nq + ch;
          vx[n][I][j] = *src;
        }
    }
  };
  if (wave * 16 < p.dvp) load_v(wave * 16);
  __syncthreads();  // lm, and w_out as seen by this workgroup
  // X = (1 + L)^-1 diag(beta) R by blocks of 16 rows, X_I = D_I^-1 (beta_I R_I - sum_{J < I} L_IJ X_J): W from the decayed
  // keys, U0 from the values. First the inverses of the diagonal blocks, one per wave, one column per lane.
  float* dinv = qh;  // [64][kDInvPitch]
  {
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      x[i] = i == i16 ? 1.f : 0.f;
#pragma unroll
      for (int s = 0; s < i; ++s) x[i] = fmaf(lm[(wave * kDSub + i) * kDPitch + wave * kDSub + s], x[s], x[i]);
    }
    if (g4 == 0)
#pragma unroll
      for (int i = 0; i < 16; ++i) dinv[(wave * kDSub + i) * kDInvPitch + i16] = x[i];
  }
  __syncthreads();
  f32x4 lo[6], di[4], be[4];
#pragma unroll
  for (int I = 0; I < 4; ++I) {
    di[I] = *(const f32x4*)&dinv[(I * kDSub + i16) * kDInvPitch + 4 * g4];
#pragma unroll
    for (int r = 0; r < 4; ++r) be[I][r] = bt[I * kDSub + 4 * g4 + r];
#pragma unroll
    for (int J = 0; J < I; ++J) lo[I * (I - 1) / 2 + J] = *(const f32x4*)&lm[(I * kDSub + i16) * kDPitch + J * kDSub + 4 * g4];
  }
  // columns in the layout of accumulators: an accumulator is the next product's right operand with the contraction
  // dealt out as 4 g + r
  auto solve = [&](auto& x) {
    constexpr int N = sizeof(x) / sizeof(x[0]);
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      f32x4 c[N];
#pragma unroll
      for (int n = 0; n < N; ++n) c[n] = x[n][I] * be[I];
#pragma unroll
      for (int J = 0; J < I; ++J)
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int n = 0; n < N; ++n) c[n] = mfma_f32(lo[I * (I - 1) / 2 + J][r], x[n][J][r], c[n]);
#pragma unroll
      for (int n = 0; n < N; ++n) x[n][I] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int n = 0; n < N; ++n) x[n][I] = mfma_f32(di[I][r], c[n][r], x[n][I]);
    }
  };
  {
    f32x4 x[NB][4];
    float* wp = w_out + (4 * g4) * DKP + wave * 16 + i16;
#pragma unroll
    for (int n = 0; n < NB; ++n)
#pragma unroll
      for (int I = 0; I < 4; ++I)
#pragma unroll
        for (int r = 0; r < 4; ++r) x[n][I][r] = wp[(I * kDSub + r) * DKP + n * 64];
    solve(x);
#pragma unroll
    for (int n = 0; n < NB; ++n)
#pragma unroll
      for (int I = 0; I < 4; ++I)
#pragma unroll
        for (int r = 0; r < 4; ++r) wp[(I * kDSub + r) * DKP + n * 64] = x[n][I][r];
  }
#pragma unroll 1
  for (int v0 = wave * 16; v0 < p.dvp; v0 += 128) {  // columns v0 .. and v0 + 64 ..
    f32x4 x[2][4];
    if (v0 != wave * 16) load_v(v0);
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      float f[TAPS];
#pragma unroll
      for (int j = 0; j < TAPS; ++j) f[j] = j >= TAPS - p.taps && v0 + 64 * n + i16 < p.dv ? T::one(vw[n][j]) : 0.f;
#pragma unroll
      for (int I = 0; I < 4; ++I) {
        float z[TAPS + 3];
#pragma unroll
        for (int j = 0; j < TAPS + 3; ++j) z[j] = chunk * kDChunk + I * kDSub + 4 * g4 - (TAPS - 1) + j >= lead ? T::one(vx[n][I][j]) : 0.f;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          float a = 0.f;
#pragma unroll
          for (int j = 0; j < TAPS; ++j) a = fmaf(f[j], z[r + j], a);
          x[n][I][r] = silu(a);
        }
      }
    }
    solve(x);
#pragma unroll
    for (int n = 0; n < 2; ++n)
      if (v0 + 64 * n < p.dvp)
#pragma unroll
        for (int I = 0; I < 4; ++I) *(f32x4*)(p.u0 + (bhc * p.dvp + v0 + 64 * n + i16) * kDChunk + I * kDSub + 4 * g4) = x[n][I];
  }
}

// 2. grid (heads * slices of 16 value columns, batch); wave w owns key rows 16 NT w .. of S (dkp = 64 NT). The slices
// of a head are `heads` workgroups apart: one XCD's L2 serves them all where the heads are a multiple of 8.
// An accumulator tile (rows 4 g + r, column lane % 16) is the B operand of the next product as it stands, with
// the contraction dealt out as 4 g + r.
template <int NT>
__global__ void __launch_bounds__(256, 1) delta_scan_kernel(const DeltaParams p) {
  __shared__ __align__(16) f32x4 xu[2][4][4][64], xo[2][4][4][64];  // [buffer][wave][row tile][lane]
  const int t = threadIdx.x, lane = t & 63, wave = __builtin_amdgcn_readfirstlane(t >> 6), g = lane >> 4, i16 = lane & 15;
  const int h = blockIdx.x % p.heads, c0 = (blockIdx.x / p.heads) * 16, b = blockIdx.y;
  const long bh = (long)b * p.heads + h;
  const int d0 = wave * NT * 16;
  float* st = p.s + bh * p.dk * p.dv;
  const bool col = c0 + i16 < p.dv;
  f32x4 s[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = d0 + 16 * i + 4 * g + r;
      const bool in = d < p.dk && col;
      const float x = st[in ? (long)d * p.dv + c0 + i16 : 0];
      s[i][r] = in ? x : 0.f;
    }
  f32x4 w[4][NT], q[4][NT], kd[4][NT], gc[NT], aq[4], u0[4];
  auto load_wq = [&](int c) {
    const float* wp = p.w + (bh * p.chunks + c) * kDChunk * p.dkp + (long)i16 * p.dkp + d0 + 4 * g;
    const float* qp = p.qe + (bh * p.chunks + c) * kDChunk * p.dkp + (long)i16 * p.dkp + d0 + 4 * g;
#pragma unroll
    for (int rt = 0; rt < 4; ++rt)
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        w[rt][i] = *(const f32x4*)(wp + (long)16 * rt * p.dkp + 16 * i);
        q[rt][i] = *(const f32x4*)(qp + (long)16 * rt * p.dkp + 16 * i);
      }
  };
  auto load_u = [&](int c) {
    const float* up = p.u0 + ((bh * p.chunks + c) * p.dvp + c0 + i16) * kDChunk + 4 * g;
#pragma unroll
    for (int j = 0; j < 4; ++j) u0[j] = *(const f32x4*)(up + 16 * j);
  };
  auto load_a = [&](int c) {
    const float* ap = p.aqk + (bh * p.chunks + c) * kDChunk * kDChunk + (long)(16 * wave + i16) * kDChunk + 4 * g;
#pragma unroll
    for (int j = 0; j < 4; ++j) aq[j] = *(const f32x4*)(ap + 16 * (j <= wave ? j : wave));
  };
  auto load_k = [&](int c) {
    const float* kp = p.kd + ((bh * p.chunks + c) * p.dkp + d0 + i16) * kDChunk + 4 * g;
#pragma unroll
    for (int i = 0; i < NT; ++i) {
#pragma unroll
      for (int j = 0; j < 4; ++j) kd[j][i] = *(const f32x4*)(kp + (long)16 * i * kDChunk + 16 * j);
      gc[i] = *(const f32x4*)(p.gc + (bh * p.chunks + c) * p.dkp + d0 + 16 * i + 4 * g);
    }
  };
  // (what the next chunk needs is requested as soon as its registers are free, and stays there)
  auto stay = [] { asm volatile("" ::: "memory"); };
  load_wq(0);
  load_u(0);
  load_a(0);
  load_k(0);
  stay();
  for (int c = 0; c < p.chunks; ++c) {
    const int buf = c & 1, next = c + 1 < p.chunks ? c + 1 : c;
    // this wave's key rows of W S and Q S
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) {
      f32x4 a = {0.f, 0.f, 0.f, 0.f}, o = a;
#pragma unroll
      for (int i = 0; i < NT; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          a = mfma_f32(w[rt][i][r], s[i][r], a);
          o = mfma_f32(q[rt][i][r], s[i][r], o);
        }
      xu[buf][wave][rt][lane] = a;
      xo[buf][wave][rt][lane] = o;
    }
    load_wq(next);
    stay();
    __syncthreads();
    f32x4 u[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const f32x4 a = xu[buf][0][j][lane], b4 = xu[buf][1][j][lane], c4 = xu[buf][2][j][lane], d4 = xu[buf][3][j][lane];
#pragma unroll
      for (int r = 0; r < 4; ++r) u[j][r] = u0[j][r] - ((a[r] + b4[r]) + (c4[r] + d4[r]));
    }
    load_u(next);
    stay();
    {
      const f32x4 a = xo[buf][0][wave][lane], b4 = xo[buf][1][wave][lane], c4 = xo[buf][2][wave][lane], d4 = xo[buf][3][wave][lane];
      f32x4 o;
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = (a[r] + b4[r]) + (c4[r] + d4[r]);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (j <= wave)
#pragma unroll
          for (int r = 0; r < 4; ++r) o = mfma_f32(aq[j][r], u[j][r], o);
      const int tk = c * kDChunk + 16 * wave + 4 * g;
      float* dst = p.o + (((long)b * p.t + tk) * p.heads + h) * p.dv + c0 + i16;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (tk + r < p.t && col) dst[(long)r * p.heads * p.dv] = o[r];
    }
    load_a(next);
    stay();
#pragma unroll
    for (int i = 0; i < NT; ++i) {
#pragma unroll
      for (int r = 0; r < 4; ++r) s[i][r] *= gc[i][r];
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) s[i] = mfma_f32(kd[j][i][r], u[j][r], s[i]);
    }
    load_k(next);
    stay();
  }
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = d0 + 16 * i + 4 * g + r;
      if (d < p.dk && col) st[(long)d * p.dv + c0 + i16] = s[i][r];
    }
}

// 3. grid (chunks, heads, batch); wave w takes tokens 16 w .. of the chunk
template <typename T>
__global__ void __launch_bounds__(256) delta_output_kernel(const DeltaParams p) {
  typedef typename T::storage S;
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, g = lane >> 4, i16 = lane & 15;
  const int chunk = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int tok0 = chunk * kDChunk + wave * kDSub;
  if (chunk == p.chunks - 1) keep_inputs<T>(p, b, h, t, 256);
  if (tok0 >= p.t) return;
  const bool vec = p.rg % 8 == 0 && p.vec;
  const int tk = tok0 + i16 < p.t ? tok0 + i16 : p.t - 1;
  const S* x = (const S*)p.proj + ((long)b * p.t + tk) * p.pitch + p.g_off;
  long at[4];  // rows of this lane
  float ss[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int tr = tok0 + 4 * g + r < p.t ? tok0 + 4 * g + r : p.t - 1;
    at[r] = (((long)b * p.t + tr) * p.heads + h) * p.dv;
  }
  for (int c0 = 0; c0 < p.dv; c0 += 64)
#pragma unroll
    for (int n = 0; n < 4; ++n) {
      const int c = c0 + 16 * n + i16;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float o = p.o[at[r] + (c < p.dv ? c : 0)];
        ss[r] = c < p.dv ? fmaf(o, o, ss[r]) : ss[r];
      }
    }
#pragma unroll
  for (int r = 0; r < 4; ++r) ss[r] = 1.f / sqrtf(row16_sum(ss[r]) / (float)p.dv + p.eps);
  for (int c0 = 0; c0 < p.dv; c0 += 64) {
    const S* wr[4];
    float gain[4], o[4][4];
    f32x4 z[4];
#pragma unroll
    for (int n = 0; n < 4; ++n) {
      const int c = c0 + 16 * n + i16, cc = c < p.dv ? c : p.dv - 1;
      wr[n] = (const S*)p.g2 + ((long)h * p.dv + cc) * p.rg;
      gain[n] = T::one(((const S*)p.gain)[cc]);
#pragma unroll
      for (int r = 0; r < 4; ++r) o[n][r] = p.o[at[r] + cc];
    }
    low_rank_tiles<T, 4>(x, wr, p.rg, vec, z);
#pragma unroll
    for (int n = 0; n < 4; ++n) {
      const int c = c0 + 16 * n + i16;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (c < p.dv && tok0 + 4 * g + r < p.t) ((S*)p.y)[at[r] + c] = T::pack(o[n][r] * ss[r] * gain[n] * sigm(z[n][r]));
    }
  }
}

// ---------------------------------------------------------------------------------------
// launchers
// ---------------------------------------------------------------------------------------
// what the chunk kernels cover
constexpr int kMaxDeltaKey = 256, kMaxDeltaTaps = 8;
static bool delta_chunked(int dk, int taps) { return dk <= kMaxDeltaKey && taps <= kMaxDeltaTaps; }
static int delta_dkp(int dk) { return dk <= 64 ? 64 : (dk <= 128 ? 128 : 256); }

// sizes whose operands the step kernel may keep in registers
static bool delta_step_held(const DeltaParams& p) {
  auto fits = [](int rows, int r) { return r % 8 == 0 && ceil_div(rows, 64) * ceil_div(r, 64) <= kLowRankHeld; };
  return p.vec && p.dv % 4 == 0 && p.taps <= 4 && fits(p.dk, p.ra) && fits(p.dv, p.rg);
}

template <typename T>
static int launch_delta_step(hipStream_t s, const DeltaParams& p) {
  int cgp = 16;
  while (cgp * 4 < p.dv) cgp <<= 1;
  if (cgp > kStepThreads || (long)p.dk * p.dv > (1L << 30)) return MUI_ERR_UNSUPPORTED;
  const int rows = ceil_div(p.dk, kStepThreads / cgp), parts = cgp <= 64 ? 8 : kStepThreads / cgp;
  const dim3 grid(p.heads, p.batch), block(kStepThreads);
  auto launch = [&](auto kernel, int nr) {
    const size_t dkp = nr > 0 ? (size_t)nr * (kStepThreads / cgp) : p.dk;
    const size_t lds = (3 * dkp + 4 * cgp + 2 * p.dv + p.ra + p.rg + 4 + (size_t)2 * parts * 4 * cgp) * 4;
    if (lds > 160 * 1024) return (int)MUI_ERR_UNSUPPORTED;
    if (lds > 48 * 1024 && hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
      return (int)MUI_ERR_LAUNCH;
    hipLaunchKernelGGL(kernel, grid, block, lds, s, p, cgp);
    return launch_status();
  };
  if constexpr (T::kDtype != MUI_DTYPE_F32) {
    if (delta_step_held(p)) {
      if (rows <= 4) return launch(delta_step_kernel<T, 4>, 4);
      if (rows <= 8) return launch(delta_step_kernel<T, 8>, 8);
      if (rows <= 16) return launch(delta_step_kernel<T, 16>, 16);
    }
  }
  return launch(delta_step_kernel<T, 0>, 0);
}

template <typename T, int NB>
static int launch_delta_chunks(hipStream_t s, const DeltaParams& p) {
  if (p.heads > 65535 || p.batch > 65535) return MUI_ERR_UNSUPPORTED;
  const size_t lds = (size_t)4 * kDChunk * kDPitch * 4;
  const dim3 grid(p.chunks, p.heads, p.batch), block(256);
  const int st = p.taps <= 4 ? launch_with_lds(delta_prepare_kernel<T, NB, 4>, grid, block, lds, s, p)
                             : launch_with_lds(delta_prepare_kernel<T, NB, kMaxDeltaTaps>, grid, block, lds, s, p);
  if (st != MUI_OK) return st;
  hipLaunchKernelGGL((delta_scan_kernel<NB>), dim3(p.heads * (p.dvp / 16), p.batch), block, 0, s, p);
  hipLaunchKernelGGL((delta_output_kernel<T>), grid, block, 0, s, p);
  return launch_status();
}

template <typename T>
static int launch_delta(hipStream_t s, const DeltaParams& p) {
  if (p.chunks == 0) return launch_delta_step<T>(s, p);
  if (p.dkp <= 64) return launch_delta_chunks<T, 1>(s, p);
  if (p.dkp <= 128) return launch_delta_chunks<T, 2>(s, p);
  return launch_delta_chunks<T, 4>(s, p);
}

// floats per (batch row, head, chunk) of the workspace, o apart
static size_t delta_unit(int dkp, int dvp) { return (size_t)kDChunk * (3 * dkp + dvp + kDChunk) + dkp; }

}  // namespace mui

using namespace mui;

extern "C" int mui_channel_delta_max_tokens(int dk, int taps) { return delta_chunked(dk, taps) ? (1 << 30) : MUI_MAX_TOKENS; }

extern "C" int mui_channel_delta_ring_rows(int taps) { return taps - 1 + MUI_MAX_TOKENS; }

extern "C" size_t mui_channel_delta_workspace_bytes(int batch, int t, int heads, int dk, int dv) {
  if (batch < 1 || t <= MUI_MAX_TOKENS || heads < 1 || dk < 1 || dk > kMaxDeltaKey || dv < 1) return 0;
  const int dkp = delta_dkp(dk), dvp = ceil_div(dv, 16) * 16;
  return ((size_t)batch * heads * ceil_div(t, kDChunk) * delta_unit(dkp, dvp) + (size_t)batch * t * heads * dv) * 4;
}

extern "C" int mui_channel_delta(mui_stream_t stream, int dtype, const mui_channel_delta_t* d, const void* proj, long pitch,
                                 float* state, void* ring, const int64_t* cache_position, const int64_t* row_start, void* y,
                                 void* workspace, int batch, int t) {
  MUI_CHECK_ARG(d && proj && state && ring && cache_position && y && batch > 0 && t > 0);
  MUI_CHECK_ARG(d->conv && d->a2 && d->dt_bias && d->a_log && d->g2 && d->gain);
  MUI_CHECK_ARG(d->heads > 0 && d->kv_heads > 0 && d->heads % d->kv_heads == 0 && d->dk > 0 && d->dv > 0 && d->ra > 0 && d->rg > 0 &&
                d->taps > 0);
  const long nq = (long)d->kv_heads * d->dk, nv = (long)d->heads * d->dv;
  MUI_CHECK_ARG(d->q_offset >= 0 && d->k_offset >= 0 && d->v_offset >= 0 && d->a_offset >= 0 && d->g_offset >= 0 && d->b_offset >= 0);
  MUI_CHECK_ARG(pitch >= d->q_offset + nq && pitch >= d->k_offset + nq && pitch >= d->v_offset + nv && pitch >= d->a_offset + d->ra &&
                pitch >= d->g_offset + d->rg && pitch >= d->b_offset + d->heads);
  if (batch > 65535 || !aligned16(state) || (long)batch * t * d->heads > (1L << 31) - 1) return MUI_ERR_UNSUPPORTED;
  DeltaParams p = {};
  p.proj = proj; p.pitch = pitch; p.q_off = d->q_offset; p.k_off = d->k_offset; p.v_off = d->v_offset; p.a_off = d->a_offset;
  p.g_off = d->g_offset; p.b_off = d->b_offset; p.conv = d->conv; p.a2 = d->a2; p.dt_bias = d->dt_bias; p.a_log = d->a_log;
  p.g2 = d->g2; p.gain = d->gain; p.q_scale = d->q_scale; p.eps = d->epsilon; p.s = state; p.ring = ring;
  p.cache_position = cache_position; p.row_start = row_start; p.y = y; p.batch = batch; p.t = t; p.heads = d->heads;
  p.kv_heads = d->kv_heads; p.dk = d->dk; p.dv = d->dv; p.ra = d->ra; p.rg = d->rg; p.taps = d->taps;
  p.vec = aligned16(proj) && aligned16(d->a2) && aligned16(d->g2) && pitch % 8 == 0 && d->a_offset % 8 == 0 && d->g_offset % 8 == 0;
  p.ring_rows = mui_channel_delta_ring_rows(d->taps); p.channels = (int)(2 * nq + nv);
  if (t > MUI_MAX_TOKENS) {
    if (!delta_chunked(d->dk, d->taps)) return MUI_ERR_UNSUPPORTED;
    MUI_CHECK_ARG(workspace);
    if (!aligned16(workspace)) return MUI_ERR_ALIGNMENT;
    p.chunks = ceil_div(t, kDChunk);
    p.dkp = delta_dkp(d->dk);
    p.dvp = ceil_div(d->dv, 16) * 16;
    const size_t units = (size_t)batch * d->heads * p.chunks;
    p.qe = (float*)workspace;
    p.w = p.qe + units * kDChunk * p.dkp;
    p.kd = p.w + units * kDChunk * p.dkp;
    p.u0 = p.kd + units * kDChunk * p.dkp;
    p.aqk = p.u0 + units * kDChunk * p.dvp;
    p.gc = p.aqk + units * kDChunk * kDChunk;
    p.o = p.gc + units * p.dkp;
  }
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MUI_DTYPE_F16) return launch_delta<F16>(s, p);
  if (dtype == MUI_DTYPE_BF16) return launch_delta<BF16>(s, p);
  if (dtype == MUI_DTYPE_F32) return launch_delta<F32>(s, p);
  return MUI_ERR_INVALID_ARG;
}
