// Mixture of experts: of E small gated feed-forwards every token uses the `top` with the largest router logits, weighted by
// the softmax over those.
//
// Router logits: products with fp32 accumulation on the matrix cores, logits kept in fp32 (an extra row may ride along: the
// gate of a shared expert).  A wave per token then takes the largest ones out one by one, in the same launch.  In a decode
// batch the routing runs beside the layer's projections, which read the same input (lr_linear_multi_route).
//
// An entry is token * top + slot; the experts' results are a row per entry, and whoever adds them to the residual weights
// and sums them (lr_residual_tanh), so nothing is added atomically and no order depends on the run.
//   up to 64 tokens   every expert's weights are streamed once, by the bands of stream_band.h with their inputs gathered:
//                     an expert's workgroups find its entries among the choices themselves, the others' leave at once
//   more              entries are sorted by expert (count, scan, scatter) and multiplied in 256-row tiles of the prefill
//                     GEMM, inputs gathered and results scattered by the entry list
// fp32: the sorted form for any number of tokens, on the fp32 tiles of residual.hip.
#include "mixer_common.h"
#include "stream_band.h"

namespace lr_detail {
int gemm_grouped(const void* x, int64_t ldx, int64_t xrows, const void* w, void* y, int64_t ldy, int N, int K, int pair_off, int64_t wstride,
                 const int32_t* tiles, const int32_t* ntiles, const int32_t* entries, int xdiv, int max_tiles, int tile_rows, hipStream_t s);   // gemm.hip
int linear_f32_grouped(const float* x, int64_t ldx, const float* w, float* y, int64_t ldy, int N, int K, const int32_t* tiles,
                       const int32_t* ntiles, const int32_t* entries, int xdiv, int max_tiles, hipStream_t s);                   // residual.hip
int linear_f32_grouped_rows();
}  // namespace lr_detail

namespace {

// ---- 16 rows per workgroup: logits router[e, :] . x[row, :] + bias[e] (rows of the router from E on have no bias), 16 ET
// router rows at a time with the columns shared out among the NW waves; then, a row per wave, the largest logits (the lower
// index among equals) and the softmax over them.  gate: sigmoid of logit E, for the shared expert.
struct Router {
  const void *x, *w, *bias;
  int64_t ldx;
  int rows, D, E, n, top;     // n: router rows, E or E + 1
  int32_t* experts;
  float *weights, *gate;
};
constexpr int EPL = 8;        // logits per lane
constexpr int router_lds_floats(int NW, int ET, int n) { return NW * ET * 256 + 16 * n; }

template <typename T, int ET, int NW>
__device__ __forceinline__ void route_rows(const Router& a, const int block, float* sm) {
  float* part = sm;                          // [NW][4 ET][64]
  float* logits = part + NW * ET * 256;      // [16][n]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g4 = lane >> 4, l16 = lane & 15;
  const int r0 = block * 16, nr = min(16, a.rows - r0), D = a.D, E = a.E, n = a.n;
  // A wave takes blocks of 128 bytes of every row, a lane 32 consecutive bytes of them in two steps (the order of the columns
  // inside a step is the same in both operands); BL blocks are in flight together.
  constexpr int V = 16 / sizeof(T), BK_ = 8 * V, BL = 4;
  constexpr int SZ = (int)sizeof(T);
  const rsrc_t rx = buffer_of(reinterpret_cast<const T*>(a.x) + (int64_t)r0 * a.ldx, (int)(((nr - 1) * a.ldx + D) * SZ));
  const int xo = l16 < nr ? (int)(l16 * a.ldx) * SZ : NOWHERE;
  for (int e0 = 0; e0 < n; e0 += 16 * ET) {
    const int ne = min(16 * ET, n - e0);
    const rsrc_t rw = buffer_of(reinterpret_cast<const T*>(a.w) + (int64_t)e0 * D, ne * D * SZ);
    f32x4_t acc[ET];
#pragma unroll
    for (int t = 0; t < ET; ++t) acc[t] = f32x4_t{0, 0, 0, 0};
    for (int k = BK_ * wave; k < D; k += BK_ * NW * BL) {
      u32x4_t xv[2 * BL], wv[2 * BL][ET];
#pragma unroll
      for (int u = 0; u < 2 * BL; ++u) {
        const int c = k + BK_ * NW * (u >> 1) + 2 * V * g4 + V * (u & 1);
        xv[u] = __builtin_amdgcn_raw_buffer_load_b128(rx, c < D && xo >= 0 ? xo + c * SZ : NOWHERE, 0, 0);
#pragma unroll
        for (int t = 0; t < ET; ++t)
          wv[u][t] = __builtin_amdgcn_raw_buffer_load_b128(rw, c < D && 16 * t + l16 < ne ? ((16 * t + l16) * D + c) * SZ : NOWHERE, 0, 0);
      }
      __builtin_amdgcn_sched_barrier(0);      // (all of them, before the first is used)
#pragma unroll
      for (int u = 0; u < 2 * BL; ++u) {
#pragma unroll
        for (int t = 0; t < ET; ++t) {
          if constexpr (sizeof(T) == 2) {
            acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, wv[u][t]), __builtin_bit_cast(bf16x8_t, xv[u]), acc[t], 0, 0, 0);
          } else {
            acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(wv[u][t][0]), __uint_as_float(xv[u][0]), acc[t], 0, 0, 0);
            acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(wv[u][t][1]), __uint_as_float(xv[u][1]), acc[t], 0, 0, 0);
            acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(wv[u][t][2]), __uint_as_float(xv[u][2]), acc[t], 0, 0, 0);
            acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(wv[u][t][3]), __uint_as_float(xv[u][3]), acc[t], 0, 0, 0);
          }
        }
      }
    }
    if (e0) __syncthreads();
#pragma unroll
    for (int t = 0; t < ET; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) part[(wave * ET * 4 + 4 * t + i) * 64 + lane] = acc[t][i];
    __syncthreads();
    // register i of tile t: router row e0 + 16 t + 4 g4 + i, row r0 + l16
    for (int o = tid; o < ET * 256; o += 64 * NW) {
      const int q = o >> 6, l = o & 63, e = e0 + 16 * (q >> 2) + 4 * (l >> 4) + (q & 3);
      if (e < n) {
        float s = 0.0f;
#pragma unroll
        for (int v = 0; v < NW; ++v) s += part[(v * ET * 4 + q) * 64 + l];
        logits[(l & 15) * n + e] = s + (e < E ? ldf(reinterpret_cast<const T*>(a.bias) + e) : 0.0f);
      }
    }
  }
  __syncthreads();
  for (int r = wave; r < nr; r += NW) {
    float* z = logits + r * n;       // (a row is one wave's: the weights take the place of the logits as they are taken out)
    float v[EPL];
#pragma unroll
    for (int i = 0; i < EPL; ++i) v[i] = lane + 64 * i < E ? z[lane + 64 * i] : -INFINITY;
    asm volatile("" ::: "memory");
    float first = 0.0f, sum = 0.0f;
    int32_t* ids = a.experts + (int64_t)(r0 + r) * a.top;
    for (int k = 0; k < a.top; ++k) {
      float m = v[0];
#pragma unroll
      for (int i = 1; i < EPL; ++i)
        if (64 * i < E) m = fmaxf(m, v[i]);
      m = wave_max(m);
      int at = -1;
#pragma unroll
      for (int i = 0; i < EPL; ++i) {
        if (64 * i < E && at < 0) {
          const unsigned long long hit = __ballot(v[i] == m && lane + 64 * i < E);
          if (hit) {
            at = 64 * i + __builtin_ctzll(hit);
            if (lane + 64 * i == at) v[i] = -INFINITY;
          }
        }
      }
      if (k == 0) first = m;
      const float w = expf(m - first);
      sum += w;
      if (lane == 0) {
        z[k] = w;
        ids[k] = at < 0 ? 0 : at;      // (at < 0: logits that are no numbers)
      }
    }
    asm volatile("" ::: "memory");     // (a wave's LDS accesses complete in order)
    for (int k = lane; k < a.top; k += 64) a.weights[(int64_t)(r0 + r) * a.top + k] = z[k] / sum;
    if (n > E && lane == 0) a.gate[r0 + r] = 1.0f / (1.0f + expf(-z[E]));
  }
}

constexpr int RW = 8;
template <typename T, int ET>
__global__ __launch_bounds__(64 * RW) void k_router(const Router a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  route_rows<T, ET, RW>(a, blockIdx.x, sm);
}

// One or two projections of a decode batch (the bands of lr_linear_multi) and its routing: the first workgroups route
template <int MT, bool XL, int ET>
__global__ __launch_bounds__(NWV * 64) void k_project_route(const Proj p0, const Proj p1, const int M, const Router a) {
  extern __shared__ __attribute__((aligned(16))) u16 sg_smem[];
  const int nr = (M + 15) / 16, id = (int)blockIdx.x - nr;
  if (id < 0) {
    route_rows<u16, ET, NWV>(a, blockIdx.x, reinterpret_cast<float*>(sg_smem));
    return;
  }
  const bool second = id >= p0.nwg;
  const Proj p = second ? p1 : p0;
  stream_band<MT, 2, false, XL>(p, M, second ? id - p0.nwg : id, sg_smem);
}

// the shared expert's activations times their gate, four values per thread
template <typename T>
__device__ __forceinline__ void gate_rows(T* s, int64_t ld, int cols, int rows, const float* __restrict__ gate, int64_t i) {
  const int quads = cols >> 2;
  const int64_t r = i / quads;
  if (r >= rows) return;
  s += r * ld + (i - r * quads) * 4;
  Quad<T> q;
  q.load(s);
  const float f = gate[r];
  float v[4];
  q.get(v);
#pragma unroll
  for (int j = 0; j < 4; ++j) v[j] *= f;
  st4(s, v);
}
template <typename T>
__global__ __launch_bounds__(256) void k_gate_rows(T* s, int64_t ld, int cols, int rows, const float* __restrict__ gate) {
  gate_rows<T>(s, ld, cols, rows, gate, (int64_t)blockIdx.x * 256 + threadIdx.x);
}

// ---- entries sorted by expert.  counts is zero on entry and left zero.
constexpr int SORT_T = 1024;
__global__ __launch_bounds__(SORT_T) void k_moe_count(const int32_t* __restrict__ experts, int n, int E, int32_t* counts) {
  extern __shared__ int32_t hist[];
  for (int e = threadIdx.x; e < E; e += SORT_T) hist[e] = 0;
  __syncthreads();
  const int i = blockIdx.x * SORT_T + threadIdx.x;
  if (i < n) atomicAdd(&hist[experts[i]], 1);
  __syncthreads();
  for (int e = threadIdx.x; e < E; e += SORT_T)
    if (hist[e]) atomicAdd(&counts[e], hist[e]);
}
// one wave: first entries, the tiles' table
__global__ __launch_bounds__(64) void k_moe_scan(int32_t* counts, int E, int tile_rows, int32_t* cursor, int32_t* tiles, int32_t* ntiles) {
  const int lane = threadIdx.x;
  int first = 0, tile = 0;
  for (int e0 = 0; e0 < E; e0 += 64) {
    const int e = e0 + lane, c = e < E ? counts[e] : 0, t = (c + tile_rows - 1) / tile_rows;
    int sc = c, st = t;
    for (int o = 1; o < 64; o <<= 1) {
      const int a = __shfl_up(sc, o, LR_WAVE), b = __shfl_up(st, o, LR_WAVE);
      if (lane >= o) { sc += a; st += b; }
    }
    if (e < E) {
      const int s0 = first + sc - c, t0 = tile + st - t;
      counts[e] = 0;
      cursor[e] = s0;
      for (int k = 0; k < t; ++k) {
        tiles[3 * (t0 + k)] = e;
        tiles[3 * (t0 + k) + 1] = s0 + k * tile_rows;
        tiles[3 * (t0 + k) + 2] = min(tile_rows, c - k * tile_rows);
      }
    }
    first += __shfl(sc, 63, LR_WAVE);
    tile += __shfl(st, 63, LR_WAVE);
  }
  if (lane == 0) *ntiles = tile;
}
__global__ __launch_bounds__(SORT_T) void k_moe_scatter(const int32_t* __restrict__ experts, int n, int E, int32_t* cursor,
                                                        int32_t* __restrict__ entries) {
  extern __shared__ int32_t hist[];      // [E] counts, then first places
  for (int e = threadIdx.x; e < E; e += SORT_T) hist[e] = 0;
  __syncthreads();
  const int i = blockIdx.x * SORT_T + threadIdx.x;
  int e = 0, r = 0;
  if (i < n) {
    e = experts[i];
    r = atomicAdd(&hist[e], 1);
  }
  __syncthreads();
  for (int k = threadIdx.x; k < E; k += SORT_T)
    if (hist[k]) hist[k] = atomicAdd(&cursor[k], hist[k]);
  __syncthreads();
  if (i < n) entries[hist[e] + r] = i;
}

// the three in one workgroup, for few entries
constexpr int SORT_ONE = 16 * SORT_T;
__global__ __launch_bounds__(SORT_T) void k_moe_sort(const int32_t* __restrict__ experts, int n, int E, int tile_rows, int32_t* __restrict__ tiles,
                                                     int32_t* __restrict__ ntiles, int32_t* __restrict__ entries) {
  extern __shared__ int32_t hist[];      // [E] counts, then next places
  const int tid = threadIdx.x;
  for (int e = tid; e < E; e += SORT_T) hist[e] = 0;
  int32_t mine[SORT_ONE / SORT_T];
#pragma unroll
  for (int j = 0; j < SORT_ONE / SORT_T; ++j) mine[j] = j * SORT_T + tid < n ? experts[j * SORT_T + tid] : -1;
  __syncthreads();
#pragma unroll
  for (int j = 0; j < SORT_ONE / SORT_T; ++j)
    if (mine[j] >= 0) atomicAdd(&hist[mine[j]], 1);
  __syncthreads();
  if (tid < 64) {
    int first = 0, tile = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int e = e0 + tid, c = e < E ? hist[e] : 0, t = (c + tile_rows - 1) / tile_rows;
      int sc = c, st = t;
      for (int o = 1; o < 64; o <<= 1) {
        const int a = __shfl_up(sc, o, LR_WAVE), b = __shfl_up(st, o, LR_WAVE);
        if (tid >= o) { sc += a; st += b; }
      }
      if (e < E) {
        const int s0 = first + sc - c, t0 = tile + st - t;
        hist[e] = s0;
        for (int k = 0; k < t; ++k) {
          tiles[3 * (t0 + k)] = e;
          tiles[3 * (t0 + k) + 1] = s0 + k * tile_rows;
          tiles[3 * (t0 + k) + 2] = min(tile_rows, c - k * tile_rows);
        }
      }
      first += __shfl(sc, 63, LR_WAVE);
      tile += __shfl(st, 63, LR_WAVE);
    }
    if (tid == 0) *ntiles = tile;
  }
  __syncthreads();
#pragma unroll
  for (int j = 0; j < SORT_ONE / SORT_T; ++j)
    if (mine[j] >= 0) entries[atomicAdd(&hist[mine[j]], 1)] = j * SORT_T + tid;
}

// ---- few tokens: one band of one expert (or, with one token, of one slot's expert).  The workgroups of the last row of the
// grid, if there is one beyond the `ny` of these, apply the shared expert's gate.
struct SharedAct {
  u16* act;
  int64_t ld;
  int cols, rows;
  const float* gate;
};
constexpr int BAND_ENTRIES = 16;      // input rows per pass over a band's weights
template <int UNITS, int KW>
__global__ __launch_bounds__(NWV * 64, 2) void k_expert_band(Proj p, const int64_t wstride, const int32_t* __restrict__ experts, const int n,
                                                          const int by_slot, const int xdiv, const int ny, const SharedAct sh) {
  extern __shared__ __attribute__((aligned(16))) u16 sg_smem[];
  int32_t* list = reinterpret_cast<int32_t*>(sg_smem + stream_band_lds_bytes<16, UNITS>() / sizeof(u16));   // [n]
  __shared__ int32_t found;
  const int tid = threadIdx.x;
  if ((int)blockIdx.y >= ny) {
    const int64_t items = (int64_t)sh.rows * (sh.cols >> 2);
    for (int64_t i = (int64_t)blockIdx.x * 256 + tid; i < items; i += (int64_t)gridDim.x * 256)
      gate_rows<u16>(sh.act, sh.ld, sh.cols, sh.rows, sh.gate, i);
    return;
  }
  int e = blockIdx.y, m = 1;
  if (by_slot) {
    e = experts[blockIdx.y];
    if (tid == 0) list[0] = blockIdx.y;
    __syncthreads();
  } else {
    if (tid < 64) {
      int c = 0;
      for (int i0 = 0; i0 < n; i0 += 64) {
        const bool hit = i0 + tid < n && experts[i0 + tid] == e;
        const unsigned long long mask = __ballot(hit);
        if (hit) list[c + __popcll(mask & ((1ull << tid) - 1))] = i0 + tid;
        c += __popcll(mask);
      }
      if (tid == 0) found = c;
    }
    __syncthreads();
    m = found;
  }
  p.w += e * wstride;
  for (int i = 0; i < m; i += BAND_ENTRIES) {
    if (i) __syncthreads();
    stream_band<16, UNITS, false, false, true, false, KW>(p, min(BAND_ENTRIES, m - i), blockIdx.x, sg_smem, list + i, xdiv);
  }
}

// KW: waves that share a band's columns (1: every wave has a band of its own, for short rows)
template <int UNITS, int KW = NWV>
int launch_band(const Proj& p, int64_t wstride, const int32_t* experts, int n, int E, bool by_slot, int xdiv, hipStream_t s, const SharedAct& sh = {}) {
  const size_t lds = stream_band_lds_bytes<16, UNITS>() + sizeof(int32_t) * n;
  static std::atomic<unsigned long long> raised{0};
  if (!lr_raise_lds_limit(reinterpret_cast<const void*>(&k_expert_band<UNITS, KW>), lds, raised)) return LR_E_LAUNCH;
  const int ny = by_slot ? n : E;
  k_expert_band<UNITS, KW><<<dim3(p.nwg, ny + (sh.act ? 1 : 0)), dim3(NWV * 64), lds, s>>>(p, wstride, experts, n, by_slot, xdiv, ny, sh);
  return lr_launch_status();
}

constexpr int BAND_ROWS = 64, BAND_LIST = 4096;      // tokens and entries up to which the bands are taken
bool by_bands(int rows, int top, int dtype) { return dtype == LR_BF16 && rows <= BAND_ROWS && (int64_t)rows * top <= BAND_LIST; }

// Height of the grouped tiles: 256 rows where experts fill them and there are tiles for most CUs.
int tile_rows(int rows, int E, int top, int I, int D, int dtype) {
  if (dtype == LR_F32) return lr_detail::linear_f32_grouped_rows();
  const int64_t n = (int64_t)rows * top, e = n < E ? n : E, tall = n / 256 + e / 2;
  return n >= 256 * e && tall * ((I + 127) / 128) >= 160 && tall * ((D + 255) / 256) >= 160 ? 256 : 128;
}
int max_tiles(int rows, int E, int top, int height) {
  const int64_t n = (int64_t)rows * top, e = n < E ? n : E;
  return (int)(n / height + e);
}

Router router_of(const lr_moe_t* d) {
  return Router{d->x, d->router, d->router_bias, d->ldx, d->rows, d->D, d->E, d->E + (d->shared ? 1 : 0), d->top, d->experts, d->weights, d->gate};
}
template <typename T, int ET>
int launch_router(const Router& a, hipStream_t s) {
  const size_t lds = sizeof(float) * router_lds_floats(RW, ET, a.n);
  static std::atomic<unsigned long long> raised{0};
  if (!lr_raise_lds_limit(reinterpret_cast<const void*>(&k_router<T, ET>), lds, raised)) return LR_E_LAUNCH;
  k_router<T, ET><<<dim3((a.rows + 15) / 16), dim3(64 * RW), lds, s>>>(a);
  return lr_launch_status();
}
template <typename T>
int route(const lr_moe_t* d, hipStream_t s) {
  const Router a = router_of(d);
  return a.n <= 16 ? launch_router<T, 1>(a, s) : a.n <= 32 ? launch_router<T, 2>(a, s) : a.n <= 48 ? launch_router<T, 3>(a, s) : launch_router<T, 4>(a, s);
}

template <int MT, bool XL, int ET>
int launch_project_route(const Proj& p0, const Proj& p1, int M, const Router& a, hipStream_t s) {
  const size_t band = stream_band_lds_bytes<MT, 2, false, XL>(), rt = sizeof(float) * router_lds_floats(NWV, ET, a.n);
  const size_t lds = band > rt ? band : rt;
  static std::atomic<unsigned long long> raised{0};
  if (!lr_raise_lds_limit(reinterpret_cast<const void*>(&k_project_route<MT, XL, ET>), lds, raised)) return LR_E_LAUNCH;
  k_project_route<MT, XL, ET><<<dim3((unsigned)((M + 15) / 16 + p0.nwg + p1.nwg)), dim3(NWV * 64), lds, s>>>(p0, p1, M, a);
  return lr_launch_status();
}
template <int ET>
int project_route(const Proj& p0, const Proj& p1, int M, const Router& a, hipStream_t s) {
  if (M > 32) return launch_project_route<64, true, ET>(p0, p1, M, a, s);
  if (M > 16) return launch_project_route<32, true, ET>(p0, p1, M, a, s);
  return M >= XLDS_M16_FROM ? launch_project_route<16, true, ET>(p0, p1, M, a, s) : launch_project_route<16, false, ET>(p0, p1, M, a, s);
}

template <typename T>
int gate(const lr_moe_t* d, hipStream_t s) {
  const int64_t items = (int64_t)d->rows * (d->shared_cols >> 2);
  k_gate_rows<T><<<dim3((unsigned)((items + 255) / 256)), dim3(256), 0, s>>>((T*)d->shared, d->ld_shared, d->shared_cols, d->rows, d->gate);
  return lr_launch_status();
}

size_t align16(size_t n) { return (n + 15) & ~(size_t)15; }

// scratch: act | (fp32) [up; gate] rows | cursor, tile count, tiles (room for the lowest ones), entries
struct Layout {
  size_t h, ints, total;
};
Layout layout(int rows, int E, int top, int I, int dtype) {
  const size_t es = dtype == LR_F32 ? 4 : 2, n = (size_t)rows * top;
  Layout l;
  l.h = align16(n * I * es);
  l.ints = l.h + (dtype == LR_F32 ? align16(n * 2 * I * es) : 0);
  l.total = l.ints + (by_bands(rows, top, dtype) ? 0 : align16(sizeof(int32_t) * ((size_t)E + 4 + 3 * (size_t)max_tiles(rows, E, top, 64) + n)));
  return l;
}

}  // namespace

extern "C" size_t lr_moe_scratch_bytes(int rows, int E, int top, int I, int dtype) {
  if (rows <= 0 || E <= 0 || top <= 0 || I <= 0 || (dtype != LR_BF16 && dtype != LR_F32)) return 0;
  return layout(rows, E, top, I, dtype).total;
}

static int check_moe(const lr_moe_t* d) {
  if (d == nullptr || d->experts == nullptr || d->weights == nullptr || d->counts == nullptr) return LR_E_NULL;
  LR_REQUIRE_PTR(d->x);
  LR_REQUIRE_PTR(d->router);
  LR_REQUIRE_PTR(d->router_bias);
  LR_REQUIRE_PTR(d->w1);
  LR_REQUIRE_PTR(d->w2);
  LR_REQUIRE_PTR(d->out);
  LR_REQUIRE_PTR(d->scratch);
  LR_OPTIONAL_PTR(d->shared);
  if (d->shared && d->gate == nullptr) return LR_E_NULL;
  if (d->dtype != LR_BF16 && d->dtype != LR_F32) return LR_E_UNSUPPORTED;
  if (d->rows <= 0 || d->D <= 0 || d->E <= 0 || d->top <= 0 || d->top > d->E || d->I <= 0 || d->ldx < d->D) return LR_E_SHAPE;
  if (d->shared && (d->shared_cols <= 0 || d->ld_shared < d->shared_cols)) return LR_E_SHAPE;
  if (d->D % 8 || d->I % 8 || d->ldx % 8 || (d->shared && (d->ld_shared % 8 || d->shared_cols % 8))) return LR_E_ALIGN;
  if (d->E > 64 * EPL || d->ldx > (1 << 24) || d->D > (1 << 22) || (int64_t)d->rows * d->top > (1 << 28)) return LR_E_UNSUPPORTED;
  return d->scratch_bytes < layout(d->rows, d->E, d->top, d->I, d->dtype).total ? LR_E_SHAPE : LR_OK;
}

extern "C" int lr_linear_multi_route(const lr_projection_t* proj, int n_proj, int M, const lr_moe_t* d, lr_stream_t stream) {
  int rc = check_moe(d);
  if (rc != LR_OK) return rc;
  if (proj == nullptr) return LR_E_NULL;
  if (n_proj < 1 || n_proj > 2 || M < 1 || M != d->rows) return LR_E_SHAPE;
  if (M > 64 || d->dtype != LR_BF16) return LR_E_UNSUPPORTED;
  Proj pr[2] = {};
  const int ncu = lr_num_cus();
  if (ncu < 1) return LR_E_LAUNCH;
  for (int i = 0; i < n_proj; ++i) {
    rc = sb_fill_projection(proj[i], pr[i]);
    if (rc != LR_OK) return rc;
    plan(pr[i], M, pr[i].pair_off ? 16 : 32, ncu);
  }
  const Router a = router_of(d);
  hipStream_t s = (hipStream_t)stream;
  return a.n <= 16 ? project_route<1>(pr[0], pr[1], M, a, s) : a.n <= 32 ? project_route<2>(pr[0], pr[1], M, a, s)
         : a.n <= 48 ? project_route<3>(pr[0], pr[1], M, a, s) : project_route<4>(pr[0], pr[1], M, a, s);
}

extern "C" int lr_moe(const lr_moe_t* d, lr_stream_t stream) {
  int rc = check_moe(d);
  if (rc != LR_OK) return rc;
  const Layout l = layout(d->rows, d->E, d->top, d->I, d->dtype);
  hipStream_t s = (hipStream_t)stream;
  char* base = reinterpret_cast<char*>(d->scratch);
  const int n = d->rows * d->top, D = d->D, I = d->I;
  void* act = base;
  if (!d->routed) {
    rc = d->dtype == LR_F32 ? route<float>(d, s) : route<u16>(d, s);
    if (rc != LR_OK) return rc;
  }
  if (d->shared && !by_bands(d->rows, d->top, d->dtype)) {
    rc = d->dtype == LR_F32 ? gate<float>(d, s) : gate<u16>(d, s);
    if (rc != LR_OK) return rc;
  }

  if (by_bands(d->rows, d->top, d->dtype)) {
    if ((int64_t)d->rows * d->ldx * 2 >= 0x7fffffff || (int64_t)n * I * 2 >= 0x7fffffff || ((int64_t)I + 64) * D * 2 >= 0x7fffffff)
      return LR_E_UNSUPPORTED;
    const bool by_slot = d->rows == 1;
    Proj p = {};
    p.x = (const u16*)d->x; p.ldx = d->ldx; p.w = (const u16*)d->w1; p.y = (u16*)act; p.ldy = I; p.N = 2 * I; p.K = D; p.pair_off = I;
    const int64_t busy = n < d->E ? n : d->E;      // experts, at most
    p.rpw = 16;
    p.nwg = (I + 15) / 16;
    const SharedAct sh = {(u16*)d->shared, d->ld_shared, d->shared_cols, d->rows, d->gate};
    rc = launch_band<2>(p, (int64_t)2 * I * D, d->experts, n, d->E, by_slot, d->top, s, sh);
    if (rc != LR_OK) return rc;
    Proj o = {};
    o.x = (const u16*)act; o.ldx = I; o.w = (const u16*)d->w2; o.y = (u16*)d->out; o.ldy = D; o.N = D; o.K = I;
    const int64_t w2 = (int64_t)I * D;
    if (I <= 1024 && busy * ((D + 127) / 128) >= 256) {
      o.rpw = 32; o.nwg = (D + 127) / 128;
      return launch_band<2, 1>(o, w2, d->experts, n, d->E, by_slot, 1, s);
    }
    if (I <= 1024 && busy * ((D + 63) / 64) >= 256) {
      o.rpw = 16; o.nwg = (D + 63) / 64;
      return launch_band<1, 1>(o, w2, d->experts, n, d->E, by_slot, 1, s);
    }
    if (busy * ((D + 31) / 32) >= 512) {
      o.rpw = 32; o.nwg = (D + 31) / 32;
      return launch_band<2>(o, w2, d->experts, n, d->E, by_slot, 1, s);
    }
    o.rpw = 16; o.nwg = (D + 15) / 16;
    return launch_band<1>(o, w2, d->experts, n, d->E, by_slot, 1, s);
  }

  const int height = tile_rows(d->rows, d->E, d->top, I, D, d->dtype), mt = max_tiles(d->rows, d->E, d->top, height);
  int32_t* cursor = reinterpret_cast<int32_t*>(base + l.ints);
  int32_t* ntiles = cursor + d->E;
  int32_t* tiles = ntiles + 4;
  int32_t* entries = tiles + 3 * (size_t)mt;
  const size_t hb = sizeof(int32_t) * d->E;
  if (n <= SORT_ONE) {
    k_moe_sort<<<dim3(1), dim3(SORT_T), hb, s>>>(d->experts, n, d->E, height, tiles, ntiles, entries);
  } else {
    const int blocks = (n + SORT_T - 1) / SORT_T;
    k_moe_count<<<dim3(blocks), dim3(SORT_T), hb, s>>>(d->experts, n, d->E, d->counts);
    k_moe_scan<<<dim3(1), dim3(64), 0, s>>>(d->counts, d->E, height, cursor, tiles, ntiles);
    k_moe_scatter<<<dim3(blocks), dim3(SORT_T), hb, s>>>(d->experts, n, d->E, cursor, entries);
  }
  if (d->dtype == LR_F32) {
    float* h = reinterpret_cast<float*>(base + l.h);
    rc = lr_detail::linear_f32_grouped((const float*)d->x, d->ldx, (const float*)d->w1, h, 2 * I, 2 * I, D, tiles, ntiles, entries, d->top, mt, s);
    if (rc != LR_OK) return rc;
    rc = lr_swiglu_f32(h, 2 * I, (float*)act, I, n, I, stream);
    if (rc != LR_OK) return rc;
    return lr_detail::linear_f32_grouped((const float*)act, I, (const float*)d->w2, (float*)d->out, D, D, I, tiles, ntiles, entries, 1, mt, s);
  }
  rc = lr_detail::gemm_grouped(d->x, d->ldx, d->rows, d->w1, act, I, I, D, I, (int64_t)2 * I * D, tiles, ntiles, entries, d->top, mt, height, s);
  if (rc != LR_OK) return rc;
  return lr_detail::gemm_grouped(act, I, n, d->w2, d->out, D, D, I, 0, (int64_t)I * D, tiles, ntiles, entries, 1, mt, height, s);
}
