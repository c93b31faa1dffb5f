// Matrix-memory recurrence (mLSTM) with exponential gating and a running maximum, per head:
//   i_t = cap tanh(ipre_t / cap),  f_t = logsigmoid(cap tanh(fpre_t / cap))
//   m_t = max(f_t + m_{t-1}, i_t),  S_t = e^{f_t + m_{t-1} - m_t} S_{t-1} + e^{i_t - m_t} k_t v_t^T,  n_t likewise with k_t
//   o_t = S_t^T q_t / (max(|n_t . q_t|, e^{-m_t}) + 1e-6)
// The state (S, n, m) and everything that enters it stays in fp32; only the projections (q, k, v) arrive in
// the activations' type.
//
//   step    (few tokens) token by token; a workgroup owns 32 value columns of a head's S. n and m are kept once
//           per such slice, so that no workgroup reads what another one writes.
//   chunks  (prompts) 64 tokens at a time: with F the running sum of f inside a chunk and a_s = i_s - F_s,
//             m_t = F_t + max(m_in, max_{s<=t} a_s)
//             S_t = e^{F_t + m_in - m_t} S_in + sum_{s<=t} e^{F_t + a_s - m_t} k_s v_s^T
//           1. every chunk's own contribution to S and n, all chunks at once
//           2. a scan over the chunks, element by element: the state each chunk starts from
//           3. every chunk's outputs, all chunks at once: (Q K^T . decays) V + decay Q S_in
//           All products are v_mfma_f32_16x16x4_f32 (A: row lane % 16, k lane / 16; B: column lane % 16;
//           D: column lane % 16, rows 4 (lane / 16) + r).
//   output  a head's o divided by its root mean square, times a gain, times sigmoid of the output gate.
// Tokens in front of a row's first slot (left padding) leave the state alone.
#include "hybrid.cuh"

namespace mui {

constexpr int kSlice = 32;    // value columns per workgroup of the step kernel
constexpr int kChunk = 64;    // tokens per chunk
constexpr float kLstmEps = 1e-6f;

struct MlstmParams {
  const void *q, *k, *v;  // token rows `pitch` apart; heads dense inside a row
  long pitch;
  const float* gates;  // [tokens, 2 heads]: i then f pre-activations
  float q_scale, cap;
  float *s, *n, *m;  // [batch, heads, dk, dv], [batch, heads, slices, dk], [batch, heads, slices]
  float* o;          // [tokens, heads, dv]
  const int64_t* cache_position;  // [t]
  const int64_t* row_start;       // [batch] or null
  int batch, t, heads, dk, dv, slices;
  // chunks
  float* cs;   // [batch, heads, chunks, dk, dv]: contribution, then state at the chunk's start
  float* cn;   // [batch, heads, chunks, dk]
  float* cg;   // [batch, heads, chunks, 4]: sum of f, m of the contribution, m at the start
  int chunks;
};

__device__ __forceinline__ bool mlstm_live(const MlstmParams& p, int b, int t) {
  return p.row_start == nullptr || p.cache_position[t] >= p.row_start[b];
}

// log gates of token t (row b), head h; a padding token neither decays nor adds
__device__ __forceinline__ void log_gates(const MlstmParams& p, int b, int t, int h, float& li, float& lf) {
  const float* g = p.gates + ((long)b * p.t + t) * 2 * p.heads;
  li = p.cap * tanhf(g[h] / p.cap);
  const float z = p.cap * tanhf(g[p.heads + h] / p.cap);
  lf = fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
  if (!mlstm_live(p, b, t)) {
    li = -INFINITY;
    lf = 0.f;
  }
}

// ---------------------------------------------------------------------------------------
// step: grid (slices, batch * heads); thread = (4 columns, one of 32 row groups)
// ---------------------------------------------------------------------------------------
extern __shared__ __align__(16) unsigned char ml_smem[];

template <typename T, bool V4>
__global__ void __launch_bounds__(256) mlstm_step_kernel(const MlstmParams p) {
  typedef typename T::storage S;
  __shared__ float red[32][kSlice + 1];
  __shared__ float nred[4];
  float* kq = (float*)ml_smem;  // k, q: dk each
  const int t = threadIdx.x, cg = t & 7, rg = t >> 3;
  const int slice = blockIdx.x, bh = blockIdx.y, b = bh / p.heads, h = bh - b * p.heads;
  const int c0 = slice * kSlice + cg * 4;
  float* st = p.s + (long)bh * p.dk * p.dv;
  float* nv = p.n + ((long)bh * p.slices + slice) * p.dk;
  float m = p.m[(long)bh * p.slices + slice];
  for (int tok = 0; tok < p.t; ++tok) {
    float* orow = p.o + (((long)b * p.t + tok) * p.heads + h) * p.dv;
    if (!mlstm_live(p, b, tok)) {  // uniform for the workgroup
      if (t < kSlice && slice * kSlice + t < p.dv) orow[slice * kSlice + t] = 0.f;
      continue;
    }
    float li, lf;
    log_gates(p, b, tok, h, li, lf);
    const float mn = fmaxf(lf + m, li), keep = expf(lf + m - mn), add = expf(li - mn);
    m = mn;
    const long base = ((long)b * p.t + tok) * p.pitch;
    float part = 0.f;
    for (int d = t; d < p.dk; d += 256) {
      const float kk = T::one(((const S*)p.k)[base + (long)h * p.dk + d]);
      const float qq = T::one(((const S*)p.q)[base + (long)h * p.dk + d]) * p.q_scale;
      kq[d] = kk;
      kq[p.dk + d] = qq;
      const float nn = fmaf(keep, nv[d], add * kk);
      nv[d] = nn;
      part = fmaf(nn, qq, part);
    }
    part = wave_sum(part);
    if ((t & 63) == 0) nred[t >> 6] = part;
    float v[4];
#pragma unroll
    for (int j = 0; j < 4; ++j)
      v[j] = c0 + j < p.dv ? add * T::one(((const S*)p.v)[base + (long)h * p.dv + c0 + j]) : 0.f;
    __syncthreads();
    float acc[4] = {0.f, 0.f, 0.f, 0.f};
    if (c0 < p.dv) {
#pragma unroll 4
      for (int d = rg; d < p.dk; d += 32) {
        float* row = st + (long)d * p.dv + c0;
        const float kk = kq[d], qq = kq[p.dk + d];
        if constexpr (V4) {
          f32x4 x = *(const f32x4*)row;
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            x[j] = fmaf(keep, x[j], kk * v[j]);
            acc[j] = fmaf(x[j], qq, acc[j]);
          }
          *(f32x4*)row = x;
        } else {
#pragma unroll
          for (int j = 0; j < 4; ++j)
            if (c0 + j < p.dv) {
              const float x = fmaf(keep, row[j], kk * v[j]);
              acc[j] = fmaf(x, qq, acc[j]);
              row[j] = x;
            }
        }
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) red[rg][cg * 4 + j] = acc[j];
    __syncthreads();
    if (t < kSlice && slice * kSlice + t < p.dv) {
      float a = 0.f;
#pragma unroll
      for (int r = 0; r < 32; ++r) a += red[r][t];
      const float nq = (nred[0] + nred[1]) + (nred[2] + nred[3]);
      orow[slice * kSlice + t] = a / (fmaxf(fabsf(nq), expf(-m)) + kLstmEps);
    }
    __syncthreads();  // kq, red, nred are free
  }
  if (t == 0) p.m[(long)bh * p.slices + slice] = m;
}

// ---------------------------------------------------------------------------------------
// chunks
// ---------------------------------------------------------------------------------------
// One wave: log gates of the chunk's 64 tokens, F = running sum of f, a = i - F, running maximum of a.
// Tokens past the end neither decay nor add. The sums are kept in double: differences of two of them
// enter exponentials, and over closed gates they grow to hundreds.
__device__ __forceinline__ void chunk_gates(const MlstmParams& p, int b, int h, int chunk, int lane, double& F, double& a,
                                            double& amax) {
  const int t = chunk * kChunk + lane;
  float li = -INFINITY, lf = 0.f;
  if (t < p.t) log_gates(p, b, t, h, li, lf);
  F = (double)lf;
#pragma unroll
  for (int d = 1; d < kWave; d <<= 1) {
    const double o = __shfl_up(F, d);
    if (lane >= d) F += o;
  }
  a = (double)li - F;
  amax = a;
#pragma unroll
  for (int d = 1; d < kWave; d <<= 1) {
    const double o = __shfl_up(amax, d);
    if (lane >= d) amax = fmax(amax, o);
  }
}

constexpr int kPitchRow = 68;  // tiles read [row][k]: 16 rows x 4 consecutive k in 64 different banks
constexpr int kPitchCol = 80;  // tiles read [k][column]: 4 rows x 16 consecutive columns likewise

// a 64 x 64 tile of a 16-bit or fp32 token-major matrix into LDS, rows past `rows` and columns past `cols` zero;
// four consecutive columns per thread and access where the rows allow it
template <typename T>
__device__ __forceinline__ void load_tile(float* dst, int pitch, const typename T::storage* src, long src_pitch, int rows,
                                          int cols, float scale) {
  typedef typename T::storage S;
  const int r0 = threadIdx.x >> 4, k = (threadIdx.x & 15) * 4;
  f32x4 v[4];
  if (((uintptr_t)src & (4 * sizeof(S) - 1)) == 0 && (src_pitch & 3) == 0 && (cols >= 64 || (cols & 3) == 0)) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {  // (clamped, not branched around)
      const bool live = r0 + 16 * i < rows && k < cols;
      const S* at = src + (live ? (long)(r0 + 16 * i) * src_pitch + k : 0);
      if constexpr (T::kDtype == MUI_DTYPE_F32) {
        v[i] = __builtin_bit_cast(f32x4, ld16(at));
      } else {
        const u32x2 w = ld8(at);
        v[i] = f32x4{T::lo(w.x), T::hi(w.x), T::lo(w.y), T::hi(w.y)};
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) v[i][j] = live ? v[i][j] * scale : 0.f;
    }
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j)
        v[i][j] = r0 + 16 * i < rows && k + j < cols ? T::one(src[(long)(r0 + 16 * i) * src_pitch + k + j]) * scale : 0.f;
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) *(f32x4*)&dst[(r0 + 16 * i) * pitch + k] = v[i];
}

// 1. contribution of a chunk: grid (chunks, heads * dk tiles * dv tiles, batch)
template <typename T>
__global__ void __launch_bounds__(256) mlstm_chunk_state_kernel(const MlstmParams p) {
  typedef typename T::storage S;
  __shared__ __align__(16) float kt[kChunk * kPitchCol], vt[kChunk * kPitchCol];
  __shared__ float w[kChunk];
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, g = lane >> 4, i16 = lane & 15;
  const int kts = (p.dk + 63) / 64, vts = (p.dv + 63) / 64;
  const int chunk = blockIdx.x, b = blockIdx.z;
  const int h = blockIdx.y / (kts * vts), tile = blockIdx.y - h * kts * vts;
  const int k0 = (tile / vts) * 64, v0 = (tile % vts) * 64;
  const long bh = (long)b * p.heads + h, bhc = bh * p.chunks + chunk;
  const int rows = p.t - chunk * kChunk < kChunk ? p.t - chunk * kChunk : kChunk;
  if (wave == 0) {
    double F, a, amax;
    chunk_gates(p, b, h, chunk, lane, F, a, amax);
    const double G = __shfl(F, 63), A = __shfl(amax, 63);
    w[lane] = A == -INFINITY ? 0.f : expf((float)(a - A));  // e^{G - F_s + i_s - (G + A)}
    if (tile == 0 && lane == 0) {
      p.cg[bhc * 4] = (float)G;
      p.cg[bhc * 4 + 1] = (float)(G + A);
    }
  }
  const long base = ((long)b * p.t + chunk * kChunk) * p.pitch;
  load_tile<T>(kt, kPitchCol, (const S*)p.k + base + (long)h * p.dk + k0, p.pitch, rows, p.dk - k0, 1.f);
  load_tile<T>(vt, kPitchCol, (const S*)p.v + base + (long)h * p.dv + v0, p.pitch, rows, p.dv - v0, 1.f);
  __syncthreads();
  f32x4 acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int s = 0; s < kChunk; s += 4) {
    const float a = kt[(s + g) * kPitchCol + wave * 16 + i16] * w[s + g];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = mfma_f32(a, vt[(s + g) * kPitchCol + 16 * j + i16], acc[j]);
  }
  float* dst = p.cs + bhc * p.dk * p.dv;
#pragma unroll
  for (int j = 0; j < 4; ++j)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = k0 + wave * 16 + 4 * g + r, c = v0 + 16 * j + i16;
      if (d < p.dk && c < p.dv) dst[(long)d * p.dv + c] = acc[j][r];
    }
  if (v0 == 0 && t < 64 && k0 + t < p.dk) {
    float a = 0.f;
    for (int s = 0; s < kChunk; ++s) a = fmaf(kt[s * kPitchCol + t], w[s], a);
    p.cn[bhc * p.dk + k0 + t] = a;
  }
}

// 2. scan over the chunks: grid (blocks of 256 elements, batch * heads); elements: dk * dv of S, then dk of n
__global__ void __launch_bounds__(256) mlstm_scan_kernel(const MlstmParams p) {
  const long bh = blockIdx.y;
  const long e = (long)blockIdx.x * 256 + threadIdx.x, ns = (long)p.dk * p.dv;
  const bool is_s = e < ns, is_n = !is_s && e < ns + p.dk;
  const float* cg = p.cg + bh * p.chunks * 4;
  float m = p.m[bh * p.slices];
  float st = 0.f;
  float* cur = nullptr;
  long step = 0;
  if (is_s) {
    st = p.s[bh * ns + e];
    cur = p.cs + bh * p.chunks * ns + e;
    step = ns;
  } else if (is_n) {
    st = p.n[bh * p.slices * p.dk + (e - ns)];
    cur = p.cn + bh * p.chunks * p.dk + (e - ns);
    step = p.dk;
  }
  for (int c0 = 0; c0 < p.chunks; c0 += 4) {
    float add[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) add[u] = cur && c0 + u < p.chunks ? cur[(c0 + u) * step] : 0.f;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int c = c0 + u;
      if (c < p.chunks) {
        const float G = cg[c * 4], ml = cg[c * 4 + 1];
        if (cur) cur[c * step] = st;
        if (e == ns) p.cg[(bh * p.chunks + c) * 4 + 2] = m;  // (the thread that owns n[0])
        const float mn = fmaxf(G + m, ml);
        st = fmaf(expf(G + m - mn), st, expf(ml - mn) * add[u]);
        m = mn;
      }
    }
  }
  if (is_s) p.s[bh * ns + e] = st;
  if (is_n)
    for (int sl = 0; sl < p.slices; ++sl) p.n[(bh * p.slices + sl) * p.dk + (e - ns)] = st;
}

// the running maximum after the last chunk, once per slice (a launch of its own: the scan's workgroups
// all read the old value)
__global__ void __launch_bounds__(64) mlstm_max_kernel(const MlstmParams p) {
  const long bh = blockIdx.x;
  const float* cg = p.cg + (bh * p.chunks + p.chunks - 1) * 4;
  const float m = fmaxf(cg[0] + cg[2], cg[1]);
  for (int i = threadIdx.x; i < p.slices; i += 64) p.m[bh * p.slices + i] = m;
}

// 3. outputs of a chunk: grid (chunks, heads * dv tiles, batch); wave w owns tokens 16 w .. of the chunk
template <typename T>
__global__ void __launch_bounds__(256) mlstm_chunk_out_kernel(const MlstmParams p) {
  typedef typename T::storage S;
  float* qt = (float*)ml_smem;                 // [64][kPitchRow] q block; later the weighted scores
  float* kt = qt + kChunk * kPitchRow;         // [64][kPitchRow] k block
  float* st = kt + kChunk * kPitchRow;         // [64][kPitchCol] state block; later v
  __shared__ double fm[kChunk], as[kChunk];  // F - m, a
  __shared__ float ms[kChunk], inter[kChunk], nq[kChunk], nb[64];
  const int t = threadIdx.x, lane = t & 63, wave = t >> 6, g = lane >> 4, i16 = lane & 15;
  const int vts = (p.dv + 63) / 64;
  const int chunk = blockIdx.x, b = blockIdx.z, h = blockIdx.y / vts, v0 = (blockIdx.y % vts) * 64;
  const long bh = (long)b * p.heads + h, bhc = bh * p.chunks + chunk;
  const int rows = p.t - chunk * kChunk < kChunk ? p.t - chunk * kChunk : kChunk;
  const float m_in = p.cg[bhc * 4 + 2];
  if (wave == 0) {
    double F, a, amax;
    chunk_gates(p, b, h, chunk, lane, F, a, amax);
    const double m = F + fmax((double)m_in, amax);
    fm[lane] = F - m;
    as[lane] = a;
    ms[lane] = (float)m;
    inter[lane] = expf((float)(F + m_in - m));
    nq[lane] = 0.f;
  }
  const long base = ((long)b * p.t + chunk * kChunk) * p.pitch;
  f32x4 sc[4], acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) sc[j] = acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < p.dk; k0 += 64) {
    __syncthreads();
    load_tile<T>(qt, kPitchRow, (const S*)p.q + base + (long)h * p.dk + k0, p.pitch, rows, p.dk - k0, p.q_scale);
    load_tile<T>(kt, kPitchRow, (const S*)p.k + base + (long)h * p.dk + k0, p.pitch, rows, p.dk - k0, 1.f);
    load_tile<F32>(st, kPitchCol, p.cs + bhc * p.dk * p.dv + (long)k0 * p.dv + v0, p.dv, p.dk - k0, p.dv - v0, 1.f);
    if (t < 64) nb[t] = k0 + t < p.dk ? p.cn[bhc * p.dk + k0 + t] : 0.f;
    __syncthreads();
    // (the state product is scaled by the tokens' decay after the loop over k)
#pragma unroll 4
    for (int k = 0; k < 64; k += 4) {
      const float a = qt[(wave * 16 + i16) * kPitchRow + k + g];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        sc[j] = mfma_f32(a, kt[(16 * j + i16) * kPitchRow + k + g], sc[j]);
        acc[j] = mfma_f32(a, st[(k + g) * kPitchCol + 16 * j + i16], acc[j]);
      }
    }
    {
      const int r = t >> 2;  // four threads per token
      float a = 0.f;
      for (int k = t & 3; k < 64; k += 4) a = fmaf(qt[r * kPitchRow + k], nb[k], a);
      a += dpp_f32<kDppXor1>(a);
      a += dpp_f32<kDppXor2>(a);
      if ((t & 3) == 0) nq[r] += a;
    }
  }
  __syncthreads();  // the q block turns into the weighted scores, the state block into v
  load_tile<T>(st, kPitchCol, (const S*)p.v + base + (long)h * p.dv + v0, p.pitch, rows, p.dv - v0, 1.f);
  float den[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int tr = wave * 16 + 4 * g + r;
    const double fmr = fm[tr];
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int s = 16 * j + i16;
      const float v = s <= tr ? sc[j][r] * expf((float)(fmr + as[s])) : 0.f;
      qt[tr * kPitchRow + s] = v;
      sum += v;
      acc[j][r] *= inter[tr];
    }
    sum = row16_sum(sum);
    den[r] = fmaxf(fabsf(sum + inter[tr] * nq[tr]), expf(-ms[tr])) + kLstmEps;
  }
  __syncthreads();
#pragma unroll 4
  for (int s = 0; s < kChunk; s += 4) {
    const float a = qt[(wave * 16 + i16) * kPitchRow + s + g];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = mfma_f32(a, st[(s + g) * kPitchCol + 16 * j + i16], acc[j]);
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int tr = wave * 16 + 4 * g + r;
    if (tr >= rows) continue;
    float* orow = p.o + (((long)b * p.t + chunk * kChunk + tr) * p.heads + h) * p.dv;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = v0 + 16 * j + i16;
      if (c < p.dv) orow[c] = acc[j][r] / den[r];
    }
  }
}

// ---------------------------------------------------------------------------------------
// output: one wave per (token, head)
// ---------------------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256) mlstm_output_kernel(const float* o, const typename T::storage* gain,
                                                           const typename T::storage* gate, long gate_pitch, float eps,
                                                           typename T::storage* y, long units, int heads, int dv) {
  const int lane = threadIdx.x & 63;
  const long u = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (u >= units) return;
  const long tok = u / heads;
  const int h = (int)(u - tok * heads);
  const float* src = o + u * dv;
  float ss = 0.f;
  for (int i = lane; i < dv; i += 64) ss = fmaf(src[i], src[i], ss);
  const float rs = rsqrtf(wave_sum(ss) / (float)dv + eps);
  for (int i = lane; i < dv; i += 64) {
    const float g = T::one(gate[tok * gate_pitch + (long)h * dv + i]);
    y[u * dv + i] = T::pack(src[i] * rs * T::one(gain[(long)h * dv + i]) / (1.f + expf(-g)));
  }
}

template <typename T>
static int launch_mlstm(hipStream_t s, const MlstmParams& p, bool chunked) {
  if (!chunked) {
    const dim3 grid(p.slices, p.batch * p.heads);
    const size_t lds = (size_t)2 * p.dk * 4;
    if (p.dv % 4 == 0 && aligned16(p.s)) return launch_with_lds(mlstm_step_kernel<T, true>, grid, dim3(256), lds, s, p);
    return launch_with_lds(mlstm_step_kernel<T, false>, grid, dim3(256), lds, s, p);
  }
  const int kts = ceil_div(p.dk, 64), vts = ceil_div(p.dv, 64);
  if ((long)p.heads * kts * vts > 65535 || p.batch > 65535) return MUI_ERR_UNSUPPORTED;
  hipLaunchKernelGGL((mlstm_chunk_state_kernel<T>), dim3(p.chunks, p.heads * kts * vts, p.batch), dim3(256), 0, s, p);
  const long elements = (long)p.dk * p.dv + p.dk;
  hipLaunchKernelGGL(mlstm_scan_kernel, dim3((unsigned)((elements + 255) / 256), p.batch * p.heads), dim3(256), 0, s, p);
  hipLaunchKernelGGL(mlstm_max_kernel, dim3(p.batch * p.heads), dim3(64), 0, s, p);
  const size_t lds = (size_t)kChunk * (2 * kPitchRow + kPitchCol) * 4;
  return launch_with_lds(mlstm_chunk_out_kernel<T>, dim3(p.chunks, p.heads * vts, p.batch), dim3(256), lds, s, p);
}

}  // namespace mui

using namespace mui;

extern "C" int mui_mlstm_slices(int dv) { return dv > 0 ? ceil_div(dv, kSlice) : 0; }

extern "C" size_t mui_mlstm_workspace_bytes(int batch, int t, int heads, int dk, int dv) {
  if (batch < 1 || t < 1 || heads < 1 || dk < 1 || dv < 1 || t <= MUI_MAX_TOKENS) return 0;
  return (size_t)batch * heads * ceil_div(t, kChunk) * ((size_t)dk * dv + dk + 4) * 4;
}

extern "C" int mui_mlstm(mui_stream_t stream, int dtype, const void* q, const void* k, const void* v, long token_pitch,
                         const float* gates, float q_scale, float gate_cap, float* state_s, float* state_n,
                         float* state_m, const int64_t* cache_position, const int64_t* row_start, float* o,
                         void* workspace, int batch, int t, int heads, int dk, int dv) {
  MUI_CHECK_ARG(q && k && v && gates && state_s && state_n && state_m && cache_position && o);
  MUI_CHECK_ARG(batch > 0 && t > 0 && heads > 0 && dk > 0 && dv > 0 && gate_cap > 0.f);
  if ((long)batch * heads > 65535) return MUI_ERR_UNSUPPORTED;
  const bool chunked = t > MUI_MAX_TOKENS;
  MUI_CHECK_ARG(!chunked || workspace);
  MlstmParams p = {};
  p.q = q; p.k = k; p.v = v; p.pitch = token_pitch; p.gates = gates; p.q_scale = q_scale; p.cap = gate_cap;
  p.s = state_s; p.n = state_n; p.m = state_m; p.o = o; p.cache_position = cache_position; p.row_start = row_start;
  p.batch = batch; p.t = t; p.heads = heads; p.dk = dk; p.dv = dv; p.slices = ceil_div(dv, kSlice);
  if (chunked) {
    p.chunks = ceil_div(t, kChunk);
    const size_t units = (size_t)batch * heads * p.chunks;
    p.cs = (float*)workspace;
    p.cn = p.cs + units * dk * dv;
    p.cg = p.cn + units * dk;
  }
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MUI_DTYPE_F16) return launch_mlstm<F16>(s, p, chunked);
  if (dtype == MUI_DTYPE_BF16) return launch_mlstm<BF16>(s, p, chunked);
  if (dtype == MUI_DTYPE_F32) return launch_mlstm<F32>(s, p, chunked);
  return MUI_ERR_INVALID_ARG;
}

extern "C" int mui_mlstm_output(mui_stream_t stream, int dtype, const float* o, const void* gain, const void* gate,
                                long gate_pitch, float epsilon, void* y, int tokens, int heads, int dv) {
  MUI_CHECK_ARG(o && gain && gate && y && tokens > 0 && heads > 0 && dv > 0);
  const long units = (long)tokens * heads;
  const dim3 grid((unsigned)((units + 3) / 4)), block(256);
  hipStream_t s = (hipStream_t)stream;
#define MUI_LAUNCH_OUT(T)                                                                                              \
  hipLaunchKernelGGL((mlstm_output_kernel<T>), grid, block, 0, s, o, (const T::storage*)gain, (const T::storage*)gate, \
                     gate_pitch, epsilon, (T::storage*)y, units, heads, dv)
  if (dtype == MUI_DTYPE_F16) MUI_LAUNCH_OUT(F16);
  else if (dtype == MUI_DTYPE_BF16) MUI_LAUNCH_OUT(BF16);
  else if (dtype == MUI_DTYPE_F32) MUI_LAUNCH_OUT(F32);
  else return MUI_ERR_INVALID_ARG;
#undef MUI_LAUNCH_OUT
  return launch_status();
}
