// Mixture of experts: of E small gated feed-forwards every token uses the `top` with the largest router logits, weighted by
// the softmax over those.
//
// Router logits: products with fp32 accumulation on the matrix cores, logits kept in fp32 (an extra row may ride along: the
// gate of a shared expert).  A wave per token then takes the largest ones out one by one.
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
                 const int32_t* tiles, const int32_t* ntiles, const int32_t* entries, int xdiv, int max_tiles, hipStream_t s);   // gemm.hip
int gemm_grouped_rows();
int linear_f32_grouped(const float* x, int64_t ldx, const float* w, float* y, int64_t ldy, int N, int K, const int32_t* tiles,
                       const int32_t* ntiles, const int32_t* entries, int xdiv, int max_tiles, hipStream_t s);                   // residual.hip
int linear_f32_grouped_rows();
}  // namespace lr_detail

namespace {

// ---- logits[row, e] = router[e, :] . x[row, :] + bias[e], fp32; 16 rows and 16 ET router rows per workgroup, its four waves
// sharing out the columns.  Rows from E on have no bias.
template <typename T, int ET>
__global__ __launch_bounds__(256) void k_router(const T* __restrict__ x, int64_t ldx, const T* __restrict__ w, const T* __restrict__ bias,
                                                float* __restrict__ logits, int rows, int D, int E, int n) {
  __shared__ float part[4][ET * 4][64];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g4 = lane >> 4, l16 = lane & 15;
  const int r0 = blockIdx.x * 16, e0 = blockIdx.y * 16 * ET;
  const T* xr = x + (int64_t)min(r0 + l16, rows - 1) * ldx;
  const T* wr[ET];
#pragma unroll
  for (int t = 0; t < ET; ++t) wr[t] = w + (int64_t)min(e0 + 16 * t + l16, n - 1) * D;
  f32x4_t acc[ET];
#pragma unroll
  for (int t = 0; t < ET; ++t) acc[t] = f32x4_t{0, 0, 0, 0};
  if constexpr (sizeof(T) == 2) {
#pragma unroll 4
    for (int k = 32 * wave; k < D; k += 128) {
      const int c = k + 8 * g4;
      const bool in = c < D;                      // (D is a multiple of 8)
      const uint4 zero = make_uint4(0, 0, 0, 0);
      const uint4 xv = in ? ld16(xr + c) : zero;
#pragma unroll
      for (int t = 0; t < ET; ++t) {
        const uint4 wv = in ? ld16(wr[t] + c) : zero;
        acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, wv), __builtin_bit_cast(bf16x8_t, xv), acc[t], 0, 0, 0);
      }
    }
  } else {
    for (int k = 16 * wave; k < D; k += 64) {
      const int c = k + 4 * g4;
      const bool in = c < D;
      const float4 zero = make_float4(0, 0, 0, 0);
      const float4 xv = in ? *reinterpret_cast<const float4*>(xr + c) : zero;
#pragma unroll
      for (int t = 0; t < ET; ++t) {
        const float4 wv = in ? *reinterpret_cast<const float4*>(wr[t] + c) : zero;
        acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(wv.x, xv.x, acc[t], 0, 0, 0);
        acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(wv.y, xv.y, acc[t], 0, 0, 0);
        acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(wv.z, xv.z, acc[t], 0, 0, 0);
        acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(wv.w, xv.w, acc[t], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int t = 0; t < ET; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) part[wave][4 * t + i][lane] = acc[t][i];
  __syncthreads();
  // register i of tile t: router row e0 + 16 t + 4 g4 + i, row r0 + l16
  for (int o = tid; o < ET * 256; o += 256) {
    const int q = o >> 6, l = o & 63, e = e0 + 16 * (q >> 2) + 4 * (l >> 4) + (q & 3), r = r0 + (l & 15);
    if (e < n && r < rows) {
      const float s = (part[0][q][l] + part[1][q][l]) + (part[2][q][l] + part[3][q][l]);
      logits[(int64_t)r * n + e] = s + (e < E ? ldf(bias + e) : 0.0f);
    }
  }
}

// ---- a wave per token: the largest logits (the lower index among equals) and the softmax over them; and the shared
// expert's activations times the sigmoid of its gate, logit E
constexpr int EPL = 8;     // logits per lane
template <typename T>
__global__ __launch_bounds__(256) void k_route(const float* __restrict__ logits, int n, int E, int top, int32_t* __restrict__ experts,
                                               float* __restrict__ weights, T* __restrict__ shared, int64_t lds_, int shared_cols, int rows) {
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (row >= rows) return;
  const float* z = logits + (int64_t)row * n;
  if (shared) {
    const float f = rcp_f(1.0f + exp2_f(-z[E] * LOG2E));
    T* s = shared + (int64_t)row * lds_;
    for (int c = lane * 4; c < shared_cols; c += 256) {
      Quad<T> q;
      q.load(s + c);
      float v[4];
      q.get(v);
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] *= f;
      st4(s + c, v);
    }
  }
  float v[EPL];
#pragma unroll
  for (int i = 0; i < EPL; ++i) v[i] = lane + 64 * i < E ? z[lane + 64 * i] : -INFINITY;
  float first = 0.0f, sum = 0.0f;
  for (int k = 0; k < top; ++k) {
    float m = v[0];
#pragma unroll
    for (int i = 1; i < EPL; ++i) m = fmaxf(m, v[i]);
    m = wave_max(m);
    int at = 0x7fffffff;
#pragma unroll
    for (int i = EPL - 1; i >= 0; --i) at = v[i] == m && lane + 64 * i < E ? lane + 64 * i : at;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) at = min(at, __shfl_xor(at, o, LR_WAVE));
    if (at >= E) at = 0;     // (no finite logit is left)
#pragma unroll
    for (int i = 0; i < EPL; ++i) v[i] = lane + 64 * i == at ? -INFINITY : v[i];
    if (k == 0) first = m;
    const float w = expf(m - first);
    sum += w;
    if (lane == 0) {
      experts[(int64_t)row * top + k] = at;
      weights[(int64_t)row * top + k] = w;
    }
  }
  if (lane == 0)
    for (int k = 0; k < top; ++k) weights[(int64_t)row * top + k] /= sum;
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

// ---- few tokens: one band of one expert (or, with one token, of one slot's expert)
constexpr int BAND_ENTRIES = 16;      // input rows per pass over a band's weights
template <int UNITS>
__global__ __launch_bounds__(NWV * 64) void k_expert_band(Proj p, const int64_t wstride, const int32_t* __restrict__ experts, const int n,
                                                          const int by_slot, const int xdiv) {
  extern __shared__ __attribute__((aligned(16))) u16 sg_smem[];
  int32_t* list = reinterpret_cast<int32_t*>(sg_smem + stream_band_lds_bytes<16, UNITS>() / sizeof(u16));   // [n]
  __shared__ int32_t found;
  const int tid = threadIdx.x;
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
    stream_band<16, UNITS, false, false, true>(p, min(BAND_ENTRIES, m - i), blockIdx.x, sg_smem, list + i, xdiv);
  }
}

template <int UNITS>
int launch_band(const Proj& p, int64_t wstride, const int32_t* experts, int n, int E, bool by_slot, int xdiv, hipStream_t s) {
  const size_t lds = stream_band_lds_bytes<16, UNITS>() + sizeof(int32_t) * n;
  static std::atomic<unsigned long long> raised{0};
  if (!lr_raise_lds_limit(reinterpret_cast<const void*>(&k_expert_band<UNITS>), lds, raised)) return LR_E_LAUNCH;
  k_expert_band<UNITS><<<dim3(p.nwg, by_slot ? n : E), dim3(NWV * 64), lds, s>>>(p, wstride, experts, n, by_slot, xdiv);
  return lr_launch_status();
}

constexpr int BAND_ROWS = 64;         // tokens up to which the bands are taken
bool by_bands(int rows, int dtype) { return dtype == LR_BF16 && rows <= BAND_ROWS; }

int tile_rows(int dtype) { return dtype == LR_F32 ? lr_detail::linear_f32_grouped_rows() : lr_detail::gemm_grouped_rows(); }
int max_tiles(int rows, int E, int top, int dtype) {
  const int64_t n = (int64_t)rows * top, e = n < E ? n : E;
  return (int)(n / tile_rows(dtype) + e);
}

template <typename T>
void router(const lr_moe_t* d, float* logits, int n, hipStream_t s) {
  const int rt = (d->rows + 15) / 16;
  if (d->rows <= 256)
    k_router<T, 1><<<dim3(rt, (n + 15) / 16), dim3(256), 0, s>>>((const T*)d->x, d->ldx, (const T*)d->router, (const T*)d->router_bias, logits,
                                                                d->rows, d->D, d->E, n);
  else
    k_router<T, 4><<<dim3(rt, (n + 63) / 64), dim3(256), 0, s>>>((const T*)d->x, d->ldx, (const T*)d->router, (const T*)d->router_bias, logits,
                                                                d->rows, d->D, d->E, n);
  k_route<T><<<dim3((d->rows + 3) / 4), dim3(256), 0, s>>>(logits, n, d->E, d->top, d->experts, d->weights, (T*)d->shared, d->ld_shared,
                                                         d->shared_cols, d->rows);
}

size_t align16(size_t n) { return (n + 15) & ~(size_t)15; }

// scratch: logits | act | (fp32) [up; gate] rows | counts, cursor, tile count, tiles, entries
struct Layout {
  size_t logits, act, h, ints, total;
};
Layout layout(int rows, int E, int top, int I, int shared, int dtype) {
  const size_t es = dtype == LR_F32 ? 4 : 2, n = (size_t)rows * top;
  Layout l;
  l.logits = 0;
  l.act = align16((size_t)rows * (E + (shared ? 1 : 0)) * sizeof(float));
  l.h = l.act + align16(n * I * es);
  l.ints = l.h + (dtype == LR_F32 ? align16(n * 2 * I * es) : 0);
  l.total = l.ints + (by_bands(rows, dtype) ? 0 : align16(sizeof(int32_t) * (2 * (size_t)E + 4 + 3 * (size_t)max_tiles(rows, E, top, dtype) + n)));
  return l;
}

}  // namespace

extern "C" size_t lr_moe_scratch_bytes(int rows, int E, int top, int I, int shared, int dtype) {
  if (rows <= 0 || E <= 0 || top <= 0 || I <= 0 || (dtype != LR_BF16 && dtype != LR_F32)) return 0;
  return layout(rows, E, top, I, shared, dtype).total;
}

extern "C" int lr_moe(const lr_moe_t* d, lr_stream_t stream) {
  if (d == nullptr || d->experts == nullptr || d->weights == nullptr || d->counts == nullptr) return LR_E_NULL;
  LR_REQUIRE_PTR(d->x);
  LR_REQUIRE_PTR(d->router);
  LR_REQUIRE_PTR(d->router_bias);
  LR_REQUIRE_PTR(d->w1);
  LR_REQUIRE_PTR(d->w2);
  LR_REQUIRE_PTR(d->out);
  LR_REQUIRE_PTR(d->scratch);
  LR_OPTIONAL_PTR(d->shared);
  if (d->dtype != LR_BF16 && d->dtype != LR_F32) return LR_E_UNSUPPORTED;
  if (d->rows <= 0 || d->D <= 0 || d->E <= 0 || d->top <= 0 || d->top > d->E || d->I <= 0 || d->ldx < d->D) return LR_E_SHAPE;
  if (d->shared && (d->shared_cols <= 0 || d->ld_shared < d->shared_cols)) return LR_E_SHAPE;
  if (d->D % 8 || d->I % 8 || d->ldx % 8 || (d->shared && (d->ld_shared % 8 || d->shared_cols % 8))) return LR_E_ALIGN;
  if (d->E > 64 * EPL || d->top > 64 || (int64_t)d->rows * d->top > (1 << 28)) return LR_E_UNSUPPORTED;
  const Layout l = layout(d->rows, d->E, d->top, d->I, d->shared != nullptr, d->dtype);
  if (d->scratch_bytes < l.total) return LR_E_SHAPE;
  hipStream_t s = (hipStream_t)stream;
  char* base = reinterpret_cast<char*>(d->scratch);
  const int n = d->rows * d->top, D = d->D, I = d->I;
  float* logits = reinterpret_cast<float*>(base + l.logits);
  void* act = base + l.act;
  const int nl = d->E + (d->shared ? 1 : 0);
  if (d->dtype == LR_F32) router<float>(d, logits, nl, s);
  else router<u16>(d, logits, nl, s);

  if (by_bands(d->rows, d->dtype)) {
    if ((int64_t)d->rows * d->ldx * 2 >= 0x7fffffff || (int64_t)n * I * 2 >= 0x7fffffff || ((int64_t)I + 64) * D * 2 >= 0x7fffffff)
      return LR_E_UNSUPPORTED;
    const bool by_slot = d->rows == 1;
    Proj p = {};
    p.x = (const u16*)d->x; p.ldx = d->ldx; p.w = (const u16*)d->w1; p.y = (u16*)act; p.ldy = I; p.N = 2 * I; p.K = D; p.pair_off = I;
    p.rpw = 16; p.nwg = (I + 15) / 16;
    int rc = launch_band<2>(p, (int64_t)2 * I * D, d->experts, n, d->E, by_slot, d->top, s);
    if (rc != LR_OK) return rc;
    Proj o = {};
    o.x = (const u16*)act; o.ldx = I; o.w = (const u16*)d->w2; o.y = (u16*)d->out; o.ldy = D; o.N = D; o.K = I;
    const int64_t busy = n < d->E ? n : d->E;
    if (busy * ((D + 31) / 32) >= 512) {
      o.rpw = 32; o.nwg = (D + 31) / 32;
      return launch_band<2>(o, (int64_t)I * D, d->experts, n, d->E, by_slot, 1, s);
    }
    o.rpw = 16; o.nwg = (D + 15) / 16;
    return launch_band<1>(o, (int64_t)I * D, d->experts, n, d->E, by_slot, 1, s);
  }

  const int mt = max_tiles(d->rows, d->E, d->top, d->dtype);
  int32_t* cursor = reinterpret_cast<int32_t*>(base + l.ints);
  int32_t* ntiles = cursor + d->E;
  int32_t* tiles = ntiles + 4;
  int32_t* entries = tiles + 3 * (size_t)mt;
  const int blocks = (n + SORT_T - 1) / SORT_T;
  const size_t hb = sizeof(int32_t) * d->E;
  k_moe_count<<<dim3(blocks), dim3(SORT_T), hb, s>>>(d->experts, n, d->E, d->counts);
  k_moe_scan<<<dim3(1), dim3(64), 0, s>>>(d->counts, d->E, tile_rows(d->dtype), cursor, tiles, ntiles);
  k_moe_scatter<<<dim3(blocks), dim3(SORT_T), hb, s>>>(d->experts, n, d->E, cursor, entries);
  if (d->dtype == LR_F32) {
    float* h = reinterpret_cast<float*>(base + l.h);
    int rc = lr_detail::linear_f32_grouped((const float*)d->x, d->ldx, (const float*)d->w1, h, 2 * I, 2 * I, D, tiles, ntiles, entries, d->top, mt, s);
    if (rc != LR_OK) return rc;
    rc = lr_swiglu_f32(h, 2 * I, (float*)act, I, n, I, stream);
    if (rc != LR_OK) return rc;
    return lr_detail::linear_f32_grouped((const float*)act, I, (const float*)d->w2, (float*)d->out, D, D, I, tiles, ntiles, entries, 1, mt, s);
  }
  const int rc = lr_detail::gemm_grouped(d->x, d->ldx, d->rows, d->w1, act, I, I, D, I, (int64_t)2 * I * D, tiles, ntiles, entries, d->top, mt, s);
  if (rc != LR_OK) return rc;
  return lr_detail::gemm_grouped(act, I, n, d->w2, d->out, D, D, I, 0, (int64_t)I * D, tiles, ntiles, entries, 1, mt, s);
}
