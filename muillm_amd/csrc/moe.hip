// Mixture-of-experts feed-forward: routing, grouping of the chosen (token, expert) pairs by expert, and
// the experts' two matrix products over the groups.
//
//   logits   fp32 [tokens, outputs]  (linear_f32 below; also the gates of recurrent layers)
//   route    s = softmax(logits); the `top` outputs with the largest s + correction are chosen, weighted
//            by their s. Outputs >= n_experts are identity experts: they take part in the choice and are
//            added by mui_moe_residual_norm, no product is computed for them.
//   group    pairs sorted by expert, cut into tiles of at most `tile_pairs` pairs of ONE expert
//   gateup   act[pair] = a(G_e x, U_e x), a(g, u) = g' sigmoid(1.702 g') (u' + 1) with g' = min(g, limit),
//            u' = clamp(u, -limit, limit)
//   down     out[pair] = D_e act[pair]
//
// Everything stays on the device (no counts travel to the host): the grids cover the largest possible
// number of tiles and workgroups without one leave at once, so a captured decode step replays whatever
// the routing does.
//
// Products, wave64 v_mfma_f32_16x16x32 (weights = A rows, pairs = B columns):
//   tile 16   up to 16 pairs of an expert: 16 gate + 16 up rows (or 32 rows) per workgroup, K dealt out to
//             its four waves, operands straight from global memory in matrix order. Decode and short
//             prompts: every chosen expert's weights are streamed once.
//   tile 128 / 256   as many pairs x as many rows, both operands through swizzled LDS stages filled by
//             LDS-direct loads; waves of 64 x 64, or of 128 x 64 with operands read a half step ahead.
// fp32 models and sizes that are no multiple of 8 take a plain one-wave-per-output kernel.
#include "skinny.cuh"

namespace mui {

enum { MOE_GATEUP = 0, MOE_DOWN = 1, MOE_F32 = 2 };

struct MoeTile { int expert, first, count, pad; };

__device__ __forceinline__ float moe_act(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.0f + __expf(-1.702f * g)) * (u + 1.0f);
}

// ---------------------------------------------------------------------------------------
// fp32 outputs of a small matrix: y[t, n] = W[n, :] . x[t, :] + bias[n], one workgroup per row
// ---------------------------------------------------------------------------------------
template <typename T, bool VEC, int TB>  // TB tokens per pass over a row
__global__ void __launch_bounds__(256) linear_f32_rows_kernel(const typename T::storage* w, const typename T::storage* x,
                                                              const typename T::storage* bias, float* y, int n, int k,
                                                              int tokens) {
  __shared__ float red[4][TB];
  const int t = threadIdx.x, row = blockIdx.x;
  const typename T::storage* wr = w + (long)row * k;
  for (int t0 = blockIdx.y * TB; t0 < tokens; t0 += gridDim.y * TB) {
    float acc[TB];
#pragma unroll
    for (int j = 0; j < TB; ++j) acc[j] = 0.f;
    if constexpr (VEC) {
#pragma unroll 2
      for (int c = t * 8; c < k; c += 256 * 8) {
        float wf[8];
        load8<T>(wr + c, wf);
#pragma unroll
        for (int j = 0; j < TB; ++j) {
          const int tk = t0 + j < tokens ? t0 + j : tokens - 1;
          float xf[8];
          load8<T>(x + (long)tk * k + c, xf);
#pragma unroll
          for (int i = 0; i < 8; ++i) acc[j] = fmaf(wf[i], xf[i], acc[j]);
        }
      }
    } else {
      for (int c = t; c < k; c += 256) {
        const float wf = T::one(wr[c]);
#pragma unroll
        for (int j = 0; j < TB; ++j) {
          const int tk = t0 + j < tokens ? t0 + j : tokens - 1;
          acc[j] = fmaf(wf, T::one(x[(long)tk * k + c]), acc[j]);
        }
      }
    }
#pragma unroll
    for (int j = 0; j < TB; ++j) {
      const float s = wave_sum(acc[j]);
      if ((t & 63) == 0) red[t >> 6][j] = s;
    }
    __syncthreads();
    if (t < TB && t0 + t < tokens)
      y[(long)(t0 + t) * n + row] = ((red[0][t] + red[1][t]) + (red[2][t] + red[3][t])) + (bias ? T::one(bias[row]) : 0.f);
    __syncthreads();
  }
}

// ---------------------------------------------------------------------------------------
// routing
// ---------------------------------------------------------------------------------------
constexpr int kMaxRouter = 1024;   // router outputs
constexpr int kRouteThreads = 1024;  // at most; few tokens take fewer
constexpr int kRouterPerLane = kMaxRouter / kWave;

// one token by one wave
template <typename T>
__device__ __forceinline__ void route_token(const float* lg, const typename T::storage* corr, int n_out, int top,
                                            int lane, int32_t* expert, float* weight, int* expert_lds = nullptr) {
  float s[kRouterPerLane], choice[kRouterPerLane];
  float mx = -INFINITY;
#pragma unroll
  for (int i = 0; i < kRouterPerLane; ++i) {
    const int e = lane + kWave * i;
    s[i] = e < n_out ? lg[e] : -INFINITY;
    mx = fmaxf(mx, s[i]);
    if (kWave * (i + 1) >= n_out) break;
  }
  mx = wave_max(mx);
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < kRouterPerLane; ++i) {
    s[i] = expf(s[i] - mx);
    sum += s[i];
    if (kWave * (i + 1) >= n_out) break;
  }
  sum = wave_sum(sum);
#pragma unroll
  for (int i = 0; i < kRouterPerLane; ++i) {
    const int e = lane + kWave * i;
    s[i] = s[i] / sum;
    choice[i] = e < n_out ? s[i] + (corr ? T::one(corr[e]) : 0.f) : -INFINITY;
    if (kWave * (i + 1) >= n_out) break;
  }
  for (int j = 0; j < top; ++j) {
    float best = -INFINITY, bs = 0.f;
    int bi = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < kRouterPerLane; ++i) {
      const int e = lane + kWave * i;
      if (choice[i] > best) { best = choice[i]; bi = e; bs = s[i]; }
      if (kWave * (i + 1) >= n_out) break;
    }
    // the wave's largest, the lowest index where several lanes hold it
    const float top_v = wave_max(best);
    uint64_t holders = __ballot(best == top_v && bi < n_out);
    int win = 0x7fffffff;
    float win_s = 0.f;
    while (holders) {
      const int l = __ffsll((unsigned long long)holders) - 1;
      const int li = __builtin_amdgcn_readlane(bi, l);
      if (li < win) {
        win = li;
        win_s = readlane_f32(bs, l);
      }
      holders &= holders - 1;
    }
    bi = win < n_out ? win : 0;  // nothing left to choose (NaN logits): stays in range
    bs = win_s;
#pragma unroll
    for (int i = 0; i < kRouterPerLane; ++i) {
      if (lane + kWave * i == bi) choice[i] = -INFINITY;
      if (kWave * (i + 1) >= n_out) break;
    }
    if (lane == 0) {
      expert[j] = bi;
      weight[j] = bs;
      if (expert_lds) expert_lds[j] = bi;
    }
  }
}

template <typename T>
__global__ void __launch_bounds__(256) moe_route_kernel(const float* logits, const typename T::storage* corr, int n_out,
                                                        int top, int tokens, int32_t* expert, float* weight) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t < tokens)
    route_token<T>(logits + (long)t * n_out, corr, n_out, top, threadIdx.x & (kWave - 1), expert + (long)t * top,
                   weight + (long)t * top);
}

// One workgroup: (ROUTE: the routing of all tokens, then) count per expert, cut into tiles, scatter.
// tiles[0].count = number of tiles, tiles[1 + i] the i-th tile; unused entries up to max_tiles get count 0.
constexpr int kChosen = 1024;
template <typename T, bool ROUTE>
__global__ void __launch_bounds__(kRouteThreads) moe_group_kernel(const float* logits, const typename T::storage* corr,
                                                                  int n_out, int n_experts, int top, int tokens,
                                                                  int tile_pairs, int max_tiles, int32_t* expert,
                                                                  float* weight, int32_t* pairs, MoeTile* tiles) {
  __shared__ int count[kMaxRouter], cursor[kMaxRouter], first_tile[kMaxRouter];
  __shared__ int n_tiles_s;
  __shared__ int chosen[ROUTE ? kChosen : 1];  // the routing's result without the way through memory
  const int t = threadIdx.x, nt_threads = blockDim.x;
  const int n_pairs = tokens * top;
  for (int e = t; e < n_experts; e += nt_threads) count[e] = 0;
  if constexpr (ROUTE) {
    for (int tk = t >> 6; tk < tokens; tk += nt_threads / kWave)
      route_token<T>(logits + (long)tk * n_out, corr, n_out, top, t & (kWave - 1), expert + (long)tk * top,
                     weight + (long)tk * top, n_pairs <= kChosen ? chosen + tk * top : nullptr);
    __threadfence_block();
  }
  auto expert_of = [&](int i) {
    if constexpr (ROUTE) return n_pairs <= kChosen ? chosen[i] : expert[i];
    else return expert[i];
  };
  __syncthreads();
  for (int i = t; i < n_pairs; i += nt_threads) {
    const int e = expert_of(i);
    if (e < n_experts) atomicAdd(&count[e], 1);
  }
  __syncthreads();
  if (t < kWave) {  // exclusive sums over experts: 64 at a time by one wave
    int pair_base = 0, tile_base = 0;
    for (int e0 = 0; e0 < n_experts; e0 += kWave) {
      const int e = e0 + t;
      const int c = e < n_experts ? count[e] : 0;
      const int nt = (c + tile_pairs - 1) / tile_pairs;
      int sc = c, st = nt;
#pragma unroll
      for (int d = 1; d < kWave; d <<= 1) {
        const int oc = __shfl_up(sc, d), ot = __shfl_up(st, d);
        if (t >= d) { sc += oc; st += ot; }
      }
      if (e < n_experts) {
        cursor[e] = pair_base + sc - c;
        first_tile[e] = tile_base + st - nt;
      }
      pair_base += __shfl(sc, kWave - 1);
      tile_base += __shfl(st, kWave - 1);
    }
    if (t == 0) n_tiles_s = tile_base < max_tiles ? tile_base : max_tiles;
  }
  __syncthreads();
  const int n_tiles = n_tiles_s;
  for (int e = t; e < n_experts; e += nt_threads) {
    const int c = count[e], base = cursor[e], ft = first_tile[e];
    for (int i = 0; i * tile_pairs < c && ft + i < max_tiles; ++i) {
      const int left = c - i * tile_pairs;
      tiles[1 + ft + i] = MoeTile{e, base + i * tile_pairs, left < tile_pairs ? left : tile_pairs, 0};
    }
  }
  for (int i = n_tiles + t; i < max_tiles; i += nt_threads) tiles[1 + i] = MoeTile{0, 0, 0, 0};
  if (t == 0) tiles[0] = MoeTile{0, 0, n_tiles, 0};
  __syncthreads();  // cursors are read above before they move
  for (int i = t; i < n_pairs; i += nt_threads) {
    const int e = expert_of(i);
    if (e < n_experts) pairs[atomicAdd(&cursor[e], 1)] = i;
  }
}

// ---------------------------------------------------------------------------------------
// products
// ---------------------------------------------------------------------------------------
struct MoeGemmParams {
  const uint16_t* w0;   // gate / down / matrix: [experts, n, k]
  const uint16_t* w1;   // up
  long expert_stride;   // elements between experts (w0 and w1)
  const uint16_t* x;    // gateup, f32: [tokens, k]; down: [pairs, k]
  const uint16_t* bias; // f32: [n] or null
  void* y;              // gateup: [pairs, n] 16-bit; down: [pairs, n] 16-bit; f32: [tokens, n] fp32
  const int32_t* pairs; // sorted pairs, null: pair i is i (f32)
  const MoeTile* tiles;
  int n, k, top, tokens;
  float limit;
  int max_tiles;
};

__device__ __forceinline__ MoeTile moe_tile_at(const MoeGemmParams& p, int i, int tile_pairs) {
  if (p.tiles) return p.tiles[1 + i];
  const int first = i * tile_pairs, left = p.tokens - first;
  return MoeTile{0, first, left < 0 ? 0 : (left < tile_pairs ? left : tile_pairs), 0};
}

// Weight rows reach LDS (a private area per wave, two stages) in runs of 256 bytes by LDS-direct loads and are
// read back as operands: 16 rows x 128 k-values per tile and stage, rows of 256 bytes whose 16-byte chunk c
// lives at chunk c ^ row. Loaded straight in operand order (64 bytes of 16 rows per instruction) the same
// bytes arrive at about two thirds of the rate.
constexpr int kT16Seg = 128;
template <typename T, int EPI>
__global__ void __launch_bounds__(256, 2) moe_tile16_kernel(const MoeGemmParams p) {
  constexpr int ROWS = EPI == MOE_GATEUP ? 16 : 32;  // outputs per workgroup
  // [wave][tile]; the stages are arrays of their own, so that the compiler can tell which loads a read waits for
  __shared__ __align__(16) uint16_t wl0[4][2][16 * kT16Seg], wl1[4][2][16 * kT16Seg];
  __shared__ int prow[16];
  const MoeTile tile = moe_tile_at(p, blockIdx.y, 16);
  if (tile.count <= 0) return;
  const int t = threadIdx.x, lane = t & (kWave - 1), wave = __builtin_amdgcn_readfirstlane(t >> 6);
  const int r16 = lane & 15, g = lane >> 4;
  const int o0 = blockIdx.x * ROWS;
  if (t < 16) {
    const int i = tile.first + (t < tile.count ? t : 0);
    prow[t] = p.pairs ? p.pairs[i] : i;
  }
  const int mine = tile.first + (r16 < tile.count ? r16 : 0);
  const int pair = p.pairs ? p.pairs[mine] : mine;
  const uint16_t* xr = p.x + (long)(EPI == MOE_GATEUP ? pair / p.top : pair) * p.k;
  const long eb = (long)tile.expert * p.expert_stride;
  // load instruction q of a tile: rows 4 q + lane / 16, this lane's logical chunk of the row
  const uint16_t* src[2][4];
  int chunk[4];
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const int r = 4 * q + g;
    chunk[q] = (r16 ^ r) * 8;
    const int ra = o0 + r < p.n ? o0 + r : p.n - 1;
    const int rb = EPI == MOE_GATEUP ? ra : (o0 + 16 + r < p.n ? o0 + 16 + r : p.n - 1);
    src[0][q] = p.w0 + eb + (long)ra * p.k;
    src[1][q] = (EPI == MOE_GATEUP ? p.w1 : p.w0) + eb + (long)rb * p.k;
  }
  f32x4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
  const int segs = (p.k + kT16Seg - 1) / kT16Seg;
  const u32x4 zero = {0u, 0u, 0u, 0u};
  // segment s into a stage (past the last one: the first again, into a stage nobody reads); chunks past
  // the end of a row read its start and meet x = 0
  auto issue = [&](int s, uint16_t (&wl)[4][2][16 * kT16Seg], u32x4 (&x)[4]) {
    const int k0 = s < segs ? s * kT16Seg : 0;
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int kk = k0 + chunk[q];
        load_lds16(src[j][q] + (kk < p.k ? kk : 0), &wl[wave][j][q * 4 * kT16Seg]);
      }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int kk = k0 + 32 * u + 8 * g;
      x[u] = ld16(xr + (kk < p.k ? kk : 0));
    }
  };
  auto multiply = [&](int s, const uint16_t (&wl)[4][2][16 * kT16Seg], const u32x4 (&x)[4]) {
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const u32x4 xv = s * kT16Seg + 32 * u + 8 * g < p.k ? x[u] : zero;
#pragma unroll
      for (int j = 0; j < 2; ++j)
        acc[j] = mfma16x16x32<T>(*(const u32x4*)&wl[wave][j][r16 * kT16Seg + ((4 * u + g) ^ r16) * 8], xv, acc[j]);
    }
  };
  u32x4 x0[4], x1[4];
  if (wave < segs) {
    issue(wave, wl0, x0);
    for (int s = wave; s < segs; s += 8) {
      issue(s + 4, wl1, x1);
      wait_loads<12>();  // everything but the newest segment has landed
      multiply(s, wl0, x0);
      if (s + 4 >= segs) break;
      issue(s + 8, wl0, x0);
      wait_loads<12>();
      multiply(s + 4, wl1, x1);
    }
  }
  wait_loads<0>();  // (no load is still on its way into LDS)
  __syncthreads();
  float(*red)[2][16][17] = (float(*)[2][16][17])wl0;
  static_assert(sizeof(wl0) >= sizeof(float) * 4 * 2 * 16 * 17, "the partial tiles fit where the weights were");
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    red[wave][0][4 * g + r][r16] = acc[0][r];
    red[wave][1][4 * g + r][r16] = acc[1][r];
  }
  __syncthreads();
  const int row = t & 15, col = t >> 4;
  float v0 = 0.f, v1 = 0.f;
#pragma unroll
  for (int w = 0; w < 4; ++w) { v0 += red[w][0][row][col]; v1 += red[w][1][row][col]; }
  if (col >= tile.count) return;
  const long out = (long)prow[col] * p.n;
  if constexpr (EPI == MOE_GATEUP) {
    if (o0 + row < p.n) ((uint16_t*)p.y)[out + o0 + row] = T::pack(moe_act(v0, v1, p.limit));
  } else if constexpr (EPI == MOE_DOWN) {
    if (o0 + row < p.n) ((uint16_t*)p.y)[out + o0 + row] = T::pack(v0);
    if (o0 + 16 + row < p.n) ((uint16_t*)p.y)[out + o0 + 16 + row] = T::pack(v1);
  } else {
    const int n0 = o0 + row, n1 = o0 + 16 + row;
    if (n0 < p.n) ((float*)p.y)[out + n0] = v0 + (p.bias ? T::one(p.bias[n0]) : 0.f);
    if (n1 < p.n) ((float*)p.y)[out + n1] = v1 + (p.bias ? T::one(p.bias[n1]) : 0.f);
  }
}

// NWR x NWT waves of 64 rows x 64 pairs each (gate/up: a wave's rows are 32 gate rows and the 32 up rows of the
// same outputs), 64 k-values per step. LDS rows are 128 bytes; 16-byte chunk c of row r lives at chunk
// c ^ ((r >> 1) & 7). DMA (k % 64 == 0): LDS-direct loads, lane i of a wave instruction fills slot i of eight
// consecutive rows, the swizzle applied to the source chunk. Otherwise the chunks go through registers and
// those past the end of a row are zeroed.
constexpr int kMgK = 64;
extern __shared__ __align__(16) unsigned char moe_smem[];

template <typename T, int EPI, bool DMA, int NWR, int NWT>
__global__ void __launch_bounds__(64 * NWR * NWT, NWR * NWT == 4 ? 2 : 1) moe_tile_kernel(const MoeGemmParams p) {
  constexpr int NW = NWR * NWT, ROWS = 64 * NWR, PAIRS = 64 * NWT, OUT = EPI == MOE_GATEUP ? ROWS / 2 : ROWS;
  constexpr int WQ = 8 / NWT, XQ = 8 / NWR;  // load instructions (eight rows each) per wave and step
  typedef uint16_t WStage[ROWS * kMgK];
  typedef uint16_t XStage[PAIRS * kMgK];
  WStage* w_lds = (WStage*)moe_smem;
  XStage* x_lds = (XStage*)(moe_smem + 2 * sizeof(WStage));
  __shared__ int prow[PAIRS];

  // tile order: a few pair tiles (of one expert, mostly) fastest, then row tiles, so that the workgroups
  // an XCD runs at a time share weight rows and token rows; the tiles are dealt to the XCDs in
  // contiguous shares of what there really is
  constexpr int SUP = PAIRS == 128 ? 4 : 2;
  const int n_tiles = p.tiles[0].count;
  const int r_tiles = (p.n + OUT - 1) / OUT;
  const int total = ((n_tiles + SUP - 1) / SUP) * SUP * r_tiles;
  const int share = (total + 7) / 8;
  const int slot = blockIdx.x >> 3, id = (blockIdx.x & 7) * share + slot;
  if (slot >= share || id >= total) return;
  const int sup = id / (SUP * r_tiles), in_sup = id - sup * SUP * r_tiles;
  const int ti = sup * SUP + in_sup % SUP;
  if (ti >= n_tiles) return;
  const MoeTile tile = p.tiles[1 + ti];
  const int o0 = (in_sup / SUP) * OUT;

  const int t = threadIdx.x, lane = t & (kWave - 1), wave = t >> 6;
  const int wr = wave / NWT, wt = wave % NWT;
  if (t < PAIRS) prow[t] = p.pairs[tile.first + (t < tile.count ? t : 0)];
  __syncthreads();
  const long eb = (long)tile.expert * p.expert_stride;
  // tile row r -> weight row
  auto wrow = [&](int r) -> const uint16_t* {
    if constexpr (EPI == MOE_GATEUP) {
      const int h = r >> 6, in = r & 63;
      int o = o0 + h * 32 + (in & 31);
      o = o < p.n ? o : p.n - 1;
      return (in >= 32 ? p.w1 : p.w0) + eb + (long)o * p.k;
    } else {
      int o = o0 + r;
      o = o < p.n ? o : p.n - 1;
      return p.w0 + eb + (long)o * p.k;
    }
  };
  // instruction q of this wave covers tile rows (q NW + wave) * 8 ..; the swizzled chunk of a row depends on
  // the lane (and the wave's parity) only
  const int sr = lane >> 3, sc = lane & 7;
  const int chunk = (sc ^ (((wave * 8 + sr) >> 1) & 7)) * 8;
  static_assert(NW % 2 == 0, "rows q NW * 8 apart share their swizzle");
  const uint16_t *wsrc[WQ], *xsrc[XQ];
#pragma unroll
  for (int q = 0; q < WQ; ++q) wsrc[q] = wrow((q * NW + wave) * 8 + sr) + chunk;
#pragma unroll
  for (int q = 0; q < XQ; ++q) {
    const int pr = prow[(q * NW + wave) * 8 + sr];
    xsrc[q] = p.x + (long)(EPI == MOE_GATEUP ? pr / p.top : pr) * p.k + chunk;
  }
  const int steps = (p.k + kMgK - 1) / kMgK;
  auto dma = [&](int s, int buf) {
#pragma unroll
    for (int q = 0; q < WQ; ++q)
      load_lds16(wsrc[q] + s * kMgK, &w_lds[buf][(q * NW + wave) * 8 * kMgK]);
#pragma unroll
    for (int q = 0; q < XQ; ++q)
      load_lds16(xsrc[q] + s * kMgK, &x_lds[buf][(q * NW + wave) * 8 * kMgK]);
  };
  u32x4 rw[WQ], rx[XQ];
  auto fetch = [&](int s) {
    const u32x4 zero = {0u, 0u, 0u, 0u};
    const bool live = s * kMgK + chunk < p.k;
    const int off = live ? s * kMgK : -chunk;
#pragma unroll
    for (int q = 0; q < WQ; ++q) { rw[q] = ld16(wsrc[q] + off); rw[q] = live ? rw[q] : zero; }
#pragma unroll
    for (int q = 0; q < XQ; ++q) { rx[q] = ld16(xsrc[q] + off); rx[q] = live ? rx[q] : zero; }
  };
  auto put = [&](int buf) {
#pragma unroll
    for (int q = 0; q < WQ; ++q) *(u32x4*)&w_lds[buf][(q * NW + wave) * 8 * kMgK + lane * 8] = rw[q];
#pragma unroll
    for (int q = 0; q < XQ; ++q) *(u32x4*)&x_lds[buf][(q * NW + wave) * 8 * kMgK + lane * 8] = rx[q];
  };
  f32x4 acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int r16 = lane & 15, lg = lane >> 4, lsw = (r16 >> 1) & 7;
  const int a_base = (wr * 64 + r16) * kMgK, b_base = (wt * 64 + r16) * kMgK;

  if constexpr (DMA) {
    dma(0, 0);
  } else {
    fetch(0);
    put(0);
  }
  for (int s = 0; s < steps; ++s) {
    const int buf = s & 1;
    const bool more = s + 1 < steps;
    if constexpr (DMA) wait_loads<0>();  // this wave's blocks of step s have landed
    __syncthreads();  // ... and everybody's; everybody is done with the other stage
    if (more) {
      if constexpr (DMA) dma(s + 1, buf ^ 1);
      else fetch(s + 1);
    }
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      u32x4 a[4], b[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) b[j] = *(const u32x4*)&x_lds[buf][b_base + j * 16 * kMgK + (((kk * 4 + lg) ^ lsw) * 8)];
#pragma unroll
      for (int i = 0; i < 4; ++i) a[i] = *(const u32x4*)&w_lds[buf][a_base + i * 16 * kMgK + (((kk * 4 + lg) ^ lsw) * 8)];
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = mfma16x16x32<T>(a[i], b[j], acc[i][j]);
    }
    if constexpr (!DMA) {
      if (more) put(buf ^ 1);
    }
  }
  // lane: pair column r16, rows 4 lg + r of every 16-row tile
  const bool n4 = (p.n & 3) == 0;
  auto store4 = [&](uint16_t* yr, int o, const float (&v)[4]) {
    if (n4 && o + 4 <= p.n) {
      *(u32x2*)&yr[o] = u32x2{T::pack2(v[0], v[1]), T::pack2(v[2], v[3])};
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (o + r < p.n) yr[o + r] = T::pack(v[r]);
    }
  };
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int c = wt * 64 + j * 16 + r16;
    if (c >= tile.count) continue;
    uint16_t* yr = (uint16_t*)p.y + (long)prow[c] * p.n;
    float v[4];
    if constexpr (EPI == MOE_GATEUP) {
#pragma unroll
      for (int i = 0; i < 2; ++i) {
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = moe_act(acc[i][j][r], acc[i + 2][j][r], p.limit);
        store4(yr, o0 + wr * 32 + i * 16 + 4 * lg, v);
      }
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = acc[i][j][r];
        store4(yr, o0 + wr * 64 + i * 16 + 4 * lg, v);
      }
    }
  }
}

// 256 rows x 256 pairs on eight waves of 128 x 64 (a quarter less LDS traffic per product than waves of 64 x 64,
// which is what bounds those), k a multiple of 64. A wave holds two sets of operands: the LDS reads of one
// half of a k-step are in flight while the other half is multiplied, and the one barrier per step has a
// half's multiplications behind it.
template <typename T, int EPI>
__global__ void __launch_bounds__(512) moe_pipe_kernel(const MoeGemmParams p) {
  constexpr int NW = 8, TILE = 256, OUT = EPI == MOE_GATEUP ? TILE / 2 : TILE, WR = 8, WT = 4;
  typedef uint16_t Stage[TILE * kMgK];
  Stage* w_lds = (Stage*)moe_smem;
  Stage* x_lds = (Stage*)(moe_smem + 2 * sizeof(Stage));
  __shared__ int prow[TILE];
  constexpr int SUP = 2;
  const int n_tiles = p.tiles[0].count;
  const int r_tiles = (p.n + OUT - 1) / OUT;
  const int total = ((n_tiles + SUP - 1) / SUP) * SUP * r_tiles;
  const int share = (total + 7) / 8;
  const int slot = blockIdx.x >> 3, id = (blockIdx.x & 7) * share + slot;
  if (slot >= share || id >= total) return;
  const int sup = id / (SUP * r_tiles), in_sup = id - sup * SUP * r_tiles;
  const int ti = sup * SUP + in_sup % SUP;
  if (ti >= n_tiles) return;
  const MoeTile tile = p.tiles[1 + ti];
  const int o0 = (in_sup / SUP) * OUT;

  const int t = threadIdx.x, lane = t & (kWave - 1), wave = __builtin_amdgcn_readfirstlane(t >> 6);
  // SIMD i runs waves i and i + 4, which are 128 pairs apart: a tile of few pairs leaves every SIMD its share
  const int wr = wave & 1, wt = wave >> 1;
  if (t < TILE) prow[t] = p.pairs[tile.first + (t < tile.count ? t : 0)];
  __syncthreads();
  // wave instruction q covers tile rows (q NW + wave) * 8 ..: 32-bit offsets from bases that are the same for
  // the wave (gate and up rows change at multiples of 64)
  const int sr = lane >> 3, sc = lane & 7;
  const int chunk = (sc ^ (((wave * 8 + sr) >> 1) & 7)) * 8;
  const uint16_t* wbase[4];
  unsigned woff[4], xoff[4];
  const long eb = (long)tile.expert * p.expert_stride;
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const int r0 = (q * NW + wave) * 8, r = r0 + sr;
    int o;
    if constexpr (EPI == MOE_GATEUP) {  // a wave's 128 rows: 64 gate rows, the 64 up rows of the same outputs
      o = o0 + (r >> 7) * 64 + (r & 63);
      wbase[q] = ((r0 & 64) ? p.w1 : p.w0) + eb;
    } else {
      o = o0 + r;
      wbase[q] = p.w0 + eb;
    }
    o = o < p.n ? o : p.n - 1;
    woff[q] = (unsigned)o * (unsigned)p.k + chunk;
    const int pr = prow[r];
    xoff[q] = (unsigned)(EPI == MOE_GATEUP ? pr / p.top : pr) * (unsigned)p.k + chunk;
  }
  auto dma = [&](int s, int buf) {
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      unsigned off = woff[q];
      asm volatile("" : "+v"(off));  // (kept as a 32-bit offset from a scalar base)
      load_lds16(wbase[q] + s * kMgK + off, &w_lds[buf][(q * NW + wave) * 8 * kMgK]);
    }
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      unsigned off = xoff[q];
      asm volatile("" : "+v"(off));
      load_lds16(p.x + s * kMgK + off, &x_lds[buf][(q * NW + wave) * 8 * kMgK]);
    }
  };
  f32x4 acc[WR][WT];
#pragma unroll
  for (int i = 0; i < WR; ++i)
#pragma unroll
    for (int j = 0; j < WT; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int r16 = lane & 15, lg = lane >> 4, lsw = (r16 >> 1) & 7;
  const int a_base = (wr * 128 + r16) * kMgK, b_base = (wt * 64 + r16) * kMgK;
  u32x4 a[2][WR], b[2][WT];
  auto read = [&](int buf, int kk, int set) {
    const int c = ((kk * 4 + lg) ^ lsw) * 8;
#pragma unroll
    for (int j = 0; j < WT; ++j) b[set][j] = *(const u32x4*)&x_lds[buf][b_base + j * 16 * kMgK + c];
#pragma unroll
    for (int i = 0; i < WR; ++i) a[set][i] = *(const u32x4*)&w_lds[buf][a_base + i * 16 * kMgK + c];
  };
  auto multiply = [&](int set) {
#pragma unroll
    for (int i = 0; i < WR; ++i)
#pragma unroll
      for (int j = 0; j < WT; ++j) acc[i][j] = mfma16x16x32<T>(a[set][i], b[set][j], acc[i][j]);
  };
  const int steps = p.k / kMgK;
  dma(0, 0);
  wait_loads<0>();
  __syncthreads();
  dma(steps > 1 ? 1 : 0, 1);
  // Loads past the last step repeat it, into a stage nobody reads any more: no branches in the loop.
  if (wt * 64 < tile.count) {
    read(0, 0, 0);
    for (int s = 0; s < steps; ++s) {
      const int buf = s & 1;
      read(buf, 1, 1);
      multiply(0);
      // issue order of the half: two matrix instructions, an LDS read, ...
#pragma unroll
      for (int i = 0; i < WR + WT; ++i) {
        __builtin_amdgcn_sched_group_barrier(0x008, 2, 0);
        __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
      }
      __builtin_amdgcn_sched_group_barrier(0x008, WR * WT - 2 * (WR + WT), 0);
      wait_loads<0>();  // step s + 1 has landed
      __syncthreads();  // ... for everybody, and everybody has read step s
      dma(s + 2 < steps ? s + 2 : steps - 1, buf);
      read(buf ^ 1, 0, 0);
      multiply(1);
      // ... a matrix instruction and a load, eight times, then two matrix instructions and a read
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        __builtin_amdgcn_sched_group_barrier(0x008, 1, 0);
        __builtin_amdgcn_sched_group_barrier(0x010, 1, 0);
      }
#pragma unroll
      for (int i = 0; i < WR + WT; ++i) {
        __builtin_amdgcn_sched_group_barrier(0x008, 2, 0);
        __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
      }
    }
  } else {  // none of this wave's pairs exist: it only keeps the loads going
    for (int s = 0; s < steps; ++s) {
      wait_loads<0>();
      __syncthreads();
      dma(s + 2 < steps ? s + 2 : steps - 1, s & 1);
    }
  }
  wait_loads<0>();  // no load is still on its way into LDS when the workgroup ends
  const bool n4 = (p.n & 3) == 0;
  auto store4 = [&](uint16_t* yr, int o, const float (&v)[4]) {
    if (n4 && o + 4 <= p.n) {
      *(u32x2*)&yr[o] = u32x2{T::pack2(v[0], v[1]), T::pack2(v[2], v[3])};
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (o + r < p.n) yr[o + r] = T::pack(v[r]);
    }
  };
#pragma unroll
  for (int j = 0; j < WT; ++j) {
    const int c = wt * 64 + j * 16 + r16;
    if (c >= tile.count) continue;
    uint16_t* yr = (uint16_t*)p.y + (long)prow[c] * p.n;
    float v[4];
    if constexpr (EPI == MOE_GATEUP) {
#pragma unroll
      for (int i = 0; i < WR / 2; ++i) {
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = moe_act(acc[i][j][r], acc[i + WR / 2][j][r], p.limit);
        store4(yr, o0 + wr * 64 + i * 16 + 4 * lg, v);
      }
    } else {
#pragma unroll
      for (int i = 0; i < WR; ++i) {
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = acc[i][j][r];
        store4(yr, o0 + wr * 128 + i * 16 + 4 * lg, v);
      }
    }
  }
}

// one wave per output of a pair: fp32 storage, and sizes that are no multiple of 8
template <typename T, int EPI>
__global__ void __launch_bounds__(256) moe_rows_kernel(const typename T::storage* w0, const typename T::storage* w1,
                                                       long expert_stride, const typename T::storage* x,
                                                       typename T::storage* y, const int32_t* expert, int n_experts,
                                                       int n, int k, int top, float limit) {
  const int lane = threadIdx.x & (kWave - 1);
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6);
  const long pair = blockIdx.y;
  if (row >= n) return;
  const int e = expert[pair];
  if (e >= n_experts) return;
  const typename T::storage* xr = x + (EPI == MOE_GATEUP ? pair / top : pair) * k;
  const typename T::storage* a = w0 + e * expert_stride + (long)row * k;
  float s0 = 0.f, s1 = 0.f;
  for (int c = lane; c < k; c += kWave) {
    const float xv = T::one(xr[c]);
    s0 = fmaf(T::one(a[c]), xv, s0);
    if constexpr (EPI == MOE_GATEUP) s1 = fmaf(T::one(w1[e * expert_stride + (long)row * k + c]), xv, s1);
  }
  s0 = wave_sum(s0);
  if constexpr (EPI == MOE_GATEUP) {
    s1 = wave_sum(s1);
    s0 = moe_act(s0, s1, limit);
  }
  if (lane == 0) y[pair * n + row] = T::pack(s0);
}

template <typename T, int EPI, int NWR, int NWT>
static int launch_moe_tile(hipStream_t s, const MoeGemmParams& p) {
  constexpr int OUT = (EPI == MOE_GATEUP ? 32 : 64) * NWR, SUP = NWT == 2 ? 4 : 2;
  const long total = (long)ceil_div(p.max_tiles, SUP) * SUP * ceil_div(p.n, OUT);
  if (total > (1L << 30)) return MUI_ERR_UNSUPPORTED;
  const dim3 grid((unsigned)((total + 7) / 8 * 8)), block(64 * NWR * NWT);
  const size_t lds = (size_t)2 * 64 * (NWR + NWT) * kMgK * 2;
  if (p.k % kMgK == 0) return launch_with_lds(moe_tile_kernel<T, EPI, true, NWR, NWT>, grid, block, lds, s, p);
  return launch_with_lds(moe_tile_kernel<T, EPI, false, NWR, NWT>, grid, block, lds, s, p);
}

template <typename T, int EPI>
static int launch_moe_product(hipStream_t s, const MoeGemmParams& p, const int32_t* expert, int n_experts, int n_pairs,
                              int tile_pairs) {
  typedef typename T::storage S;
  bool rows = T::kDtype == MUI_DTYPE_F32 || p.k % 8 != 0 || tile_pairs == 0;
  rows = rows || !aligned16(p.w0) || (p.w1 && !aligned16(p.w1)) || !aligned16(p.x) || p.expert_stride % 8 != 0;
  if (rows) {
    // pairs are one dimension of the grid: whole tokens' worth of them per launch
    const int step = 65535 / p.top * p.top;
    if (step < 1) return MUI_ERR_UNSUPPORTED;
    for (int first = 0; first < n_pairs; first += step) {
      const int cnt = n_pairs - first < step ? n_pairs - first : step;
      const long xrow = EPI == MOE_GATEUP ? first / p.top : first;
      hipLaunchKernelGGL((moe_rows_kernel<T, EPI>), dim3(ceil_div(p.n, 4), cnt), dim3(256), 0, s, (const S*)p.w0,
                         (const S*)p.w1, p.expert_stride, (const S*)p.x + xrow * p.k, (S*)p.y + (long)first * p.n,
                         expert + first, n_experts, p.n, p.k, p.top, p.limit);
    }
    return launch_status();
  }
  if constexpr (T::kDtype != MUI_DTYPE_F32) {
    if (tile_pairs == 16) {
      if (p.max_tiles > 65535) return MUI_ERR_UNSUPPORTED;
      hipLaunchKernelGGL((moe_tile16_kernel<T, EPI>), dim3(ceil_div(p.n, EPI == MOE_GATEUP ? 16 : 32), p.max_tiles),
                         dim3(256), 0, s, p);
      return launch_status();
    }
    if (((uintptr_t)p.y & 7) != 0) return MUI_ERR_ALIGNMENT;
    if (tile_pairs == 128) return launch_moe_tile<T, EPI, 2, 2>(s, p);
    if (tile_pairs == 256) {
      const long xrows = EPI == MOE_GATEUP ? p.tokens : (long)p.tokens * p.top;
      if (p.k % kMgK == 0 && (long)p.n * p.k < (1L << 30) && xrows * p.k < (1L << 30)) {
        const long total = (long)ceil_div(p.max_tiles, 2) * 2 * ceil_div(p.n, EPI == MOE_GATEUP ? 128 : 256);
        if (total > (1L << 30)) return MUI_ERR_UNSUPPORTED;
        return launch_with_lds(moe_pipe_kernel<T, EPI>, dim3((unsigned)((total + 7) / 8 * 8)), dim3(512),
                               (size_t)4 * 256 * kMgK * 2, s, p);
      }
      return launch_moe_tile<T, EPI, 4, 4>(s, p);
    }
    return MUI_ERR_INVALID_ARG;
  }
  return MUI_ERR_UNSUPPORTED;
}

template <typename T>
static int launch_linear_f32(hipStream_t s, const void* w, const void* x, const void* bias, float* y, int n, int k,
                             int tokens) {
  typedef typename T::storage S;
  const bool vec = k % 8 == 0 && aligned16(w) && aligned16(x);
  if constexpr (T::kDtype != MUI_DTYPE_F32) {
    if (vec && tokens > MUI_MAX_TOKENS) {
      MoeGemmParams p = {};
      p.w0 = (const uint16_t*)w; p.x = (const uint16_t*)x; p.bias = (const uint16_t*)bias; p.y = y; p.n = n; p.k = k;
      p.top = 1; p.tokens = tokens;
      const int tiles = ceil_div(tokens, 16);
      if (tiles > 65535) return MUI_ERR_UNSUPPORTED;
      hipLaunchKernelGGL((moe_tile16_kernel<T, MOE_F32>), dim3(ceil_div(n, 32), tiles), dim3(256), 0, s, p);
      return launch_status();
    }
  }
  auto launch = [&](auto kernel, int tb) {
    int ty = ceil_div(tokens, tb);
    if (ty > 4096) ty = 4096;
    hipLaunchKernelGGL(kernel, dim3(n, ty), dim3(256), 0, s, (const S*)w, (const S*)x, (const S*)bias, y, n, k, tokens);
    return launch_status();
  };
  if (!vec) return launch(linear_f32_rows_kernel<T, false, 4>, 4);
  if (tokens == 1) return launch(linear_f32_rows_kernel<T, true, 1>, 1);
  return launch(linear_f32_rows_kernel<T, true, 4>, 4);
}

template <typename T>
static int launch_route(hipStream_t s, const float* logits, const void* corr, int n_out, int n_experts, int top,
                        int tokens, int tile_pairs, int max_tiles, int32_t* expert, float* weight, int32_t* pairs,
                        MoeTile* tiles) {
  typedef typename T::storage S;
  const bool one = tokens <= 64 && tile_pairs;
  if (!one)
    hipLaunchKernelGGL((moe_route_kernel<T>), dim3(ceil_div(tokens, 4)), dim3(256), 0, s, logits, (const S*)corr, n_out,
                       top, tokens, expert, weight);
  if (!tile_pairs) return launch_status();
  if (one)
    hipLaunchKernelGGL((moe_group_kernel<T, true>), dim3(1), dim3(tokens <= 4 ? 256 : kRouteThreads), 0, s, logits, (const S*)corr, n_out,
                       n_experts, top, tokens, tile_pairs, max_tiles, expert, weight, pairs, tiles);
  else
    hipLaunchKernelGGL((moe_group_kernel<T, false>), dim3(1), dim3(kRouteThreads), 0, s, logits, (const S*)corr, n_out,
                       n_experts, top, tokens, tile_pairs, max_tiles, expert, weight, pairs, tiles);
  return launch_status();
}

}  // namespace mui

using namespace mui;

#define MUI_BY_DTYPE(call)                                  \
  do {                                                      \
    if (dtype == MUI_DTYPE_F16) { typedef F16 TT; return call; }   \
    if (dtype == MUI_DTYPE_BF16) { typedef BF16 TT; return call; } \
    if (dtype == MUI_DTYPE_F32) { typedef F32 TT; return call; }   \
    return MUI_ERR_INVALID_ARG;                             \
  } while (0)

extern "C" int mui_linear_f32(mui_stream_t stream, int dtype, const void* weights, const void* x, const void* bias,
                              float* y, int n_out, int k_in, int tokens) {
  MUI_CHECK_ARG(weights && x && y && n_out > 0 && k_in > 0 && tokens > 0);
  MUI_BY_DTYPE((launch_linear_f32<TT>((hipStream_t)stream, weights, x, bias, y, n_out, k_in, tokens)));
}

extern "C" int mui_moe_tile_pairs(int dtype, int tokens, int top, int n_experts, int width, int ff) {
  if (dtype == MUI_DTYPE_F32 || width % 8 || ff % 8 || n_experts < 1) return 0;
  // 16-pair tiles stream an expert's weights once per tile; from about a dozen pairs per expert on a wide tile
  // is cheaper even half empty. Of the two widths the one whose tiles cost less (a 256-pair tile, rarely full,
  // about 1.3 times as much as a 128-pair one).
  const long per = (long)tokens * top / n_experts;
  if (per < 12) return 16;
  return 13 * ((per + 255) / 256) < 10 * ((per + 127) / 128) ? 256 : 128;
}

extern "C" int mui_moe_max_tiles(int tokens, int top, int n_experts, int tile_pairs) {
  if (tile_pairs < 1) return 0;
  const long pairs = (long)tokens * top;
  return (int)(pairs / tile_pairs + (pairs < n_experts ? pairs : n_experts));
}

extern "C" int mui_moe_route(mui_stream_t stream, int dtype, const float* logits, const void* correction, int n_experts,
                             int n_identity, int top, int tokens, int tile_pairs, int32_t* expert, float* weight,
                             int32_t* pairs, void* tiles) {
  MUI_CHECK_ARG(logits && expert && weight && tokens > 0 && n_experts >= 0 && n_identity >= 0);
  const int n_out = n_experts + n_identity;
  MUI_CHECK_ARG(n_out > 0 && top > 0 && top <= n_out);
  MUI_CHECK_ARG(tile_pairs == 0 || tile_pairs == 16 || tile_pairs == 128 || tile_pairs == 256);
  MUI_CHECK_ARG(tile_pairs == 0 || (pairs && tiles));
  if (n_out > kMaxRouter || (long)tokens * top > (1L << 30)) return MUI_ERR_UNSUPPORTED;
  const int mt = mui_moe_max_tiles(tokens, top, n_experts, tile_pairs);
  MUI_BY_DTYPE((launch_route<TT>((hipStream_t)stream, logits, correction, n_out, n_experts, top, tokens, tile_pairs, mt,
                                 expert, weight, pairs, (MoeTile*)tiles)));
}

extern "C" int mui_moe_gateup(mui_stream_t stream, int dtype, const void* gate, const void* up, long expert_stride,
                              const void* x, float limit, const int32_t* expert, const int32_t* pairs,
                              const void* tiles, int tile_pairs, void* act, int n_experts, int n_inter, int k_in,
                              int top, int tokens) {
  MUI_CHECK_ARG(gate && up && x && expert && act && n_experts > 0 && n_inter > 0 && k_in > 0 && top > 0 && tokens > 0);
  MUI_CHECK_ARG(tile_pairs == 0 || (pairs && tiles));
  MoeGemmParams p = {};
  p.w0 = (const uint16_t*)gate; p.w1 = (const uint16_t*)up; p.expert_stride = expert_stride; p.x = (const uint16_t*)x;
  p.y = act; p.pairs = pairs; p.tiles = (const MoeTile*)tiles; p.n = n_inter; p.k = k_in; p.top = top; p.tokens = tokens;
  p.limit = limit; p.max_tiles = mui_moe_max_tiles(tokens, top, n_experts, tile_pairs);
  MUI_BY_DTYPE((launch_moe_product<TT, MOE_GATEUP>((hipStream_t)stream, p, expert, n_experts, tokens * top, tile_pairs)));
}

extern "C" int mui_moe_down(mui_stream_t stream, int dtype, const void* down, long expert_stride, const void* act,
                            const int32_t* expert, const int32_t* pairs, const void* tiles, int tile_pairs, void* out,
                            int n_experts, int n_out, int k_in, int top, int tokens) {
  MUI_CHECK_ARG(down && act && expert && out && n_experts > 0 && n_out > 0 && k_in > 0 && top > 0 && tokens > 0);
  MUI_CHECK_ARG(tile_pairs == 0 || (pairs && tiles));
  MoeGemmParams p = {};
  p.w0 = (const uint16_t*)down; p.expert_stride = expert_stride; p.x = (const uint16_t*)act; p.y = out; p.pairs = pairs;
  p.tiles = (const MoeTile*)tiles; p.n = n_out; p.k = k_in; p.top = top; p.tokens = tokens;
  p.max_tiles = mui_moe_max_tiles(tokens, top, n_experts, tile_pairs);
  MUI_BY_DTYPE((launch_moe_product<TT, MOE_DOWN>((hipStream_t)stream, p, expert, n_experts, tokens * top, tile_pairs)));
}
