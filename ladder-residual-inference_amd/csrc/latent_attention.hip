// Sliding-window attention over a low-rank latent: the cache holds one normalised latent c [rank] per token, per head
// k = W_uk c and v = W_uv c; position i sees positions i - window + 1 .. i.
//
// Prompt portions expand the latents of the window and the portion into k and v (lr_latent_window gathers them, the
// caller's linear expands them) and attend there: on the matrix cores (attention.hip) where the head sizes allow it, one
// wave per query otherwise.
// Single tokens and the shortest portions never form k and v: q is taken through W_uk once, scores and sums run on the
// latents, and the result goes through W_uv (lr_latent_attention).  Scores, softmax and sums are fp32.
#include "mixer_common.h"

namespace lr_detail {
int window_attention_mfma(const lr_window_attention_t* d, lr_stream_t stream);   // attention.hip
}

namespace {

// one wave per row: the latent's norm, into the cache at the row's position
template <typename T>
__global__ __launch_bounds__(256) void k_latent_update(const T* __restrict__ c, int64_t ld, const T* __restrict__ gain,
                                                       const int32_t* __restrict__ pos, T* __restrict__ cache, int rows,
                                                       int S, int rank, int ldc, int Smax, float eps, int32_t* err) {
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (row >= rows) return;
  const int b = row / S, s = row - b * S;
  const int p = pos[s];
  if (p < 0 || p >= Smax) {
    if (err && lane == 0) *err = LR_DEV_POS_RANGE;
    return;
  }
  const T* src = c + (int64_t)row * ld;
  float ss = 0.0f;
  for (int r = lane; r < rank; r += 64) {
    const float f = ldf(src + r);
    ss += f * f;
  }
  ss = wave_sum(ss);
  const float inv = 1.0f / sqrtf(ss / (float)rank + eps);
  T* dst = cache + ((int64_t)b * Smax + p) * ldc;
  for (int r = lane; r < ldc; r += 64) stf(dst + r, r < rank ? ldf(src + r) * inv * ldf(gain + r) : 0.0f);
}

__global__ __launch_bounds__(256) void k_latent_window(const uint4* __restrict__ cache, const int32_t* __restrict__ pos,
                                                       uint4* __restrict__ out, int n, int window, int q16, int Smax) {
  const int b = blockIdx.y;
  const int i = blockIdx.x * 256 + threadIdx.x;   // 16-byte piece of this sequence's n rows
  if (i >= n * q16) return;
  const int row = i / q16;
  const int p = lr_window_base(pos[0], window, n, Smax) + row;
  out[(int64_t)b * n * q16 + i] = p >= 0 && p < Smax ? cache[((int64_t)b * Smax + p) * q16 + (i - row * q16)]
                                                     : make_uint4(0, 0, 0, 0);
}

struct WinAttn {
  const void* q;
  int64_t ldq, hq;          // row stride, head stride
  const void *k, *v;
  int64_t kb, kr, kh, vb, vr, vh;   // strides of a sequence, a key row, a head
  void* y;
  int64_t ldy, hy;
  const int32_t* pos;
  int S, H, dk, dv, window, n_keys, windowed_rows, Smax;
  float scale;
};

// One wave per (query, head, sequence): 64 keys at a time, a lane per key for the scores, a lane per dimension for the
// sums; running maximum and sum.  Any sizes up to 1024 value dimensions, any storage types.
template <typename TQ, typename TK, typename TO>
__global__ __launch_bounds__(64) void k_window_attention(const WinAttn a) {
  extern __shared__ __attribute__((aligned(16))) float qs[];   // [dk] then [64] weights
  float* ps = qs + ((a.dk + 3) & ~3);
  const int h = blockIdx.x, s = blockIdx.y, b = blockIdx.z, lane = threadIdx.x;
  const int64_t row = (int64_t)b * a.S + s;
  const int p = a.pos[s];
  const int base = a.windowed_rows ? lr_window_base(a.pos[0], a.window, a.n_keys, a.Smax) : 0;
  const TQ* q = reinterpret_cast<const TQ*>(a.q) + row * a.ldq + h * a.hq;
  for (int d = lane; d < a.dk; d += 64) qs[d] = ldf(q + d);
  __syncthreads();
  const TK* kb = reinterpret_cast<const TK*>(a.k) + b * a.kb + h * a.kh;
  const TK* vb = reinterpret_cast<const TK*>(a.v) + b * a.vb + h * a.vh;
  constexpr int DV = 16;
  float acc[DV];
#pragma unroll
  for (int i = 0; i < DV; ++i) acc[i] = 0.0f;
  float m = -INFINITY, l = 0.0f;
  const int lo = max(0, p - a.window + 1), hi = min(p, base + a.n_keys - 1);
  for (int j0 = lo; j0 <= hi; j0 += 64) {
    const int j = j0 + lane;
    float sc = -INFINITY;
    if (j <= hi) {
      const TK* kr = kb + (int64_t)(j - base) * a.kr;
      sc = 0.0f;
      for (int d = 0; d < a.dk; ++d) sc = fmaf(qs[d], ldf(kr + d), sc);
      sc *= a.scale;
    }
    const float mn = fmaxf(m, wave_max(sc));
    const float corr = expf(m - mn), w = expf(sc - mn);   // first round: m = -inf, corr = 0
    l = l * corr + wave_sum(w);
    m = mn;
    __syncthreads();
    ps[lane] = w;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < DV; ++i) acc[i] *= corr;
    const int nj = min(64, hi - j0 + 1);
    for (int jj = 0; jj < nj; ++jj) {
      const TK* vr = vb + (int64_t)(j0 + jj - base) * a.vr;
      const float wj = ps[jj];
#pragma unroll
      for (int i = 0; i < DV; ++i)
        if (lane + 64 * i < a.dv) acc[i] = fmaf(wj, ldf(vr + lane + 64 * i), acc[i]);
    }
  }
  const float inv = l > 0.0f ? 1.0f / l : 0.0f;
  TO* y = reinterpret_cast<TO*>(a.y) + row * a.ldy + h * a.hy;
#pragma unroll
  for (int i = 0; i < DV; ++i)
    if (lane + 64 * i < a.dv) stf(y + lane + 64 * i, acc[i] * inv);
}

// q' [rows, H, ldr] fp32: q' = W_uk^T q per head
template <typename T>
__global__ __launch_bounds__(256) void k_latent_absorb(const T* __restrict__ q, int64_t ldq, const T* __restrict__ uk,
                                                       float* __restrict__ out, int H, int dk, int ldr) {
  extern __shared__ float qs[];
  const int h = blockIdx.x;
  const int64_t row = blockIdx.y;
  for (int d = threadIdx.x; d < dk; d += 256) qs[d] = ldf(q + row * ldq + h * dk + d);
  __syncthreads();
  for (int r = threadIdx.x; r < ldr; r += 256) {
    float acc = 0.0f;
    const T* w = uk + (int64_t)h * dk * ldr + r;
#pragma unroll 8
    for (int d = 0; d < dk; ++d) acc = fmaf(qs[d], ldf(w + (int64_t)d * ldr), acc);
    out[(row * H + h) * ldr + r] = acc;
  }
}

// y[row, h dv + e] = W_uv[h dv + e, :] . o[row, h, :]
template <typename T>
__global__ __launch_bounds__(256) void k_latent_up(const float* __restrict__ o, const T* __restrict__ uv, T* __restrict__ y,
                                                   int64_t ldy, int H, int dv, int ldr) {
  extern __shared__ float os[];
  const int h = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int64_t row = blockIdx.y;
  for (int r = threadIdx.x; r < ldr; r += 256) os[r] = o[(row * H + h) * ldr + r];
  __syncthreads();
  for (int e = wave; e < dv; e += 4) {
    const T* w = uv + ((int64_t)h * dv + e) * ldr;
    float acc = 0.0f;
    for (int r = lane; r < ldr; r += 64) acc = fmaf(ldf(w + r), os[r], acc);
    acc = wave_sum(acc);
    if (lane == 0) stf(y + row * ldy + h * dv + e, acc);
  }
}

template <typename TQ, typename TK, typename TO>
int launch_window(const WinAttn& a, int B, hipStream_t s) {
  const size_t lds = sizeof(float) * (((a.dk + 3) & ~3) + 64);
  k_window_attention<TQ, TK, TO><<<dim3(a.H, a.S, B), dim3(64), lds, s>>>(a);
  return lr_launch_status();
}

template <typename T>
int latent_attention(const lr_latent_attention_t* d, hipStream_t s) {
  float* qa = reinterpret_cast<float*>(d->scratch);
  const int rows = d->B * d->S;
  float* ol = qa + (size_t)rows * d->H * d->ldr;
  k_latent_absorb<T><<<dim3(d->H, rows), dim3(256), d->dk * sizeof(float), s>>>((const T*)d->q, d->ldq, (const T*)d->uk, qa,
                                                                               d->H, d->dk, d->ldr);
  WinAttn a = {};
  a.q = qa; a.ldq = (int64_t)d->H * d->ldr; a.hq = d->ldr;
  a.k = a.v = d->cache;
  a.kb = a.vb = (int64_t)d->Smax * d->ldr; a.kr = a.vr = d->ldr; a.kh = a.vh = 0;
  a.y = ol; a.ldy = a.ldq; a.hy = d->ldr; a.pos = d->pos;
  a.S = d->S; a.H = d->H; a.dk = a.dv = d->ldr; a.window = d->window; a.n_keys = d->Smax; a.Smax = d->Smax;
  a.scale = d->scale;
  const int rc = launch_window<float, T, float>(a, d->B, s);
  if (rc != LR_OK) return rc;
  k_latent_up<T><<<dim3(d->H, rows), dim3(256), d->ldr * sizeof(float), s>>>(ol, (const T*)d->uv, (T*)d->y, d->ldy, d->H,
                                                                            d->dv, d->ldr);
  return lr_launch_status();
}

}  // namespace

extern "C" int lr_latent_update(const void* c, int64_t ld, const void* gain, const int32_t* pos, void* cache, int B, int S,
                                int rank, int ldc, int Smax, float eps, int dtype, int32_t* err, lr_stream_t stream) {
  if (c == nullptr || pos == nullptr) return LR_E_NULL;
  LR_REQUIRE_PTR(gain);
  LR_REQUIRE_PTR(cache);
  if (B <= 0 || S <= 0 || rank <= 0 || ldc < rank || Smax <= 0 || ld < rank || (int64_t)B * S > 0x7fffffff) return LR_E_SHAPE;
  if (ldc % 8) return LR_E_ALIGN;
  const int rows = B * S;
  const dim3 grid((rows + 3) / 4), blk(256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == LR_BF16)
    k_latent_update<u16><<<grid, blk, 0, s>>>((const u16*)c, ld, (const u16*)gain, pos, (u16*)cache, rows, S, rank, ldc,
                                              Smax, eps, err);
  else if (dtype == LR_F32)
    k_latent_update<float><<<grid, blk, 0, s>>>((const float*)c, ld, (const float*)gain, pos, (float*)cache, rows, S, rank,
                                                ldc, Smax, eps, err);
  else
    return LR_E_UNSUPPORTED;
  return lr_launch_status();
}

extern "C" int lr_latent_window(const void* cache, const int32_t* pos, void* rows, int B, int n, int window, int ldc,
                                int Smax, int dtype, lr_stream_t stream) {
  LR_REQUIRE_PTR(cache);
  LR_REQUIRE_PTR(rows);
  if (pos == nullptr) return LR_E_NULL;
  if (B <= 0 || B > 65535 || n <= 0 || n > Smax || window <= 0 || ldc <= 0) return LR_E_SHAPE;
  if (ldc % 8) return LR_E_ALIGN;
  if (dtype != LR_BF16 && dtype != LR_F32) return LR_E_UNSUPPORTED;
  const int q16 = ldc * (dtype == LR_F32 ? 4 : 2) / 16;
  if ((int64_t)n * q16 > 0x7fffff00) return LR_E_UNSUPPORTED;
  k_latent_window<<<dim3((unsigned)(((int64_t)n * q16 + 255) / 256), B), dim3(256), 0, (hipStream_t)stream>>>(
      (const uint4*)cache, pos, (uint4*)rows, n, window, q16, Smax);
  return lr_launch_status();
}

extern "C" int lr_window_attention(const lr_window_attention_t* d, lr_stream_t stream) {
  if (d == nullptr || d->q == nullptr || d->k == nullptr || d->v == nullptr || d->y == nullptr || d->pos == nullptr)
    return LR_E_NULL;
  if (d->B <= 0 || d->S <= 0 || d->H <= 0 || d->dk <= 0 || d->dv <= 0 || d->window <= 0 || d->n_keys <= 0 ||
      d->n_keys > d->Smax)
    return LR_E_SHAPE;
  if (d->ldq < (int64_t)d->H * d->dk || d->ldy < (int64_t)d->H * d->dv || d->ldk < (int64_t)d->H * d->dk ||
      d->ldk < (int64_t)d->H * d->dv)
    return LR_E_SHAPE;
  if (d->B > 65535) return LR_E_UNSUPPORTED;
  {
    const int rc = lr_detail::window_attention_mfma(d, stream);
    if (rc != LR_E_UNSUPPORTED) return rc;
  }
  if (d->S > 65535) return LR_E_UNSUPPORTED;
  if (d->dv > 1024 || d->dk > 8192) return LR_E_UNSUPPORTED;
  WinAttn a = {};
  a.q = d->q; a.ldq = d->ldq; a.hq = d->dk;
  a.k = d->k; a.kb = (int64_t)d->n_keys * d->ldk; a.kr = d->ldk; a.kh = d->dk;
  a.v = d->v; a.vb = a.kb; a.vr = d->ldk; a.vh = d->dv;
  a.y = d->y; a.ldy = d->ldy; a.hy = d->dv; a.pos = d->pos;
  a.S = d->S; a.H = d->H; a.dk = d->dk; a.dv = d->dv; a.window = d->window; a.n_keys = d->n_keys; a.windowed_rows = 1;
  a.Smax = d->Smax; a.scale = d->scale;
  hipStream_t s = (hipStream_t)stream;
  if (d->dtype == LR_BF16) return launch_window<u16, u16, u16>(a, d->B, s);
  if (d->dtype == LR_F32) return launch_window<float, float, float>(a, d->B, s);
  return LR_E_UNSUPPORTED;
}

extern "C" size_t lr_latent_attention_scratch_bytes(int B, int S, int H, int ldr, int Smax) {
  if (B <= 0 || S <= 0 || H <= 0 || ldr <= 0 || Smax <= 0) return 0;
  return (size_t)2 * B * S * H * ldr * sizeof(float);
}

extern "C" int lr_latent_attention(const lr_latent_attention_t* d, lr_stream_t stream) {
  if (d == nullptr || d->q == nullptr || d->y == nullptr || d->pos == nullptr) return LR_E_NULL;
  LR_REQUIRE_PTR(d->uk);
  LR_REQUIRE_PTR(d->uv);
  LR_REQUIRE_PTR(d->cache);
  LR_REQUIRE_PTR(d->scratch);
  if (d->B <= 0 || d->S <= 0 || d->H <= 0 || d->dk <= 0 || d->dv <= 0 || d->ldr <= 0 || d->window <= 0 || d->Smax <= 0)
    return LR_E_SHAPE;
  if (d->ldq < (int64_t)d->H * d->dk || d->ldy < (int64_t)d->H * d->dv) return LR_E_SHAPE;
  if (d->scratch_bytes < lr_latent_attention_scratch_bytes(d->B, d->S, d->H, d->ldr, d->Smax)) return LR_E_SHAPE;
  if (d->ldr % 8) return LR_E_ALIGN;
  if (d->ldr > 1024 || (int64_t)d->B * d->S > 65535) return LR_E_UNSUPPORTED;
  if (d->dtype == LR_BF16) return latent_attention<u16>(d, (hipStream_t)stream);
  if (d->dtype == LR_F32) return latent_attention<float>(d, (hipStream_t)stream);
  return LR_E_UNSUPPORTED;
}
