// Sliding-window attention over a low-rank latent: the cache holds one normalised latent c [rank] per token, per head
// k = W_uk c and v = W_uv c; position i sees positions i - window + 1 .. i.
//
// Prompt portions expand the latents of the window and the portion into k and v (lr_latent_window gathers them, the
// caller's linear expands them) and attend there: on the matrix cores (attention.hip) where the head sizes allow it, one
// wave per query otherwise.
// Single tokens and the shortest portions never form k and v: q is taken through W_uk once, scores and sums run on the
// latents -- on the matrix cores, the keys cut into ranges that run side by side --, and the merged result goes through
// W_uv (lr_latent_attention: three launches, the cache write included).  Scores, softmax and sums are fp32.
#include "mixer_common.h"

namespace lr_detail {
int window_attention_mfma(const lr_window_attention_t* d, lr_stream_t stream);   // attention.hip
}

namespace {

// a wave: the latent of one row, normed, into the cache at the row's position
template <typename T>
__device__ __forceinline__ void latent_row(const T* __restrict__ c, int64_t ld, const T* __restrict__ gain,
                                           const int32_t* __restrict__ pos, T* __restrict__ cache, int row, int S, int rank,
                                           int ldc, int Smax, float eps, int32_t* err) {
  const int lane = threadIdx.x & 63;
  const int b = row / S, s = row - b * S;
  const int p = pos[s];
  if (p < 0 || p >= Smax) {
    if (err && lane == 0) *err = LR_DEV_POS_RANGE;
    return;
  }
  const T* src = c + (int64_t)row * ld;
  T* dst = cache + ((int64_t)b * Smax + p) * ldc;
  // 1024 columns at a time, all of a lane's loads in flight together
  float ss = 0.0f;
  constexpr int N = 16;
  T x[N], g[N];
  auto load = [&](int c0) {
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const int j = c0 + i * 64 + lane;
      x[i] = src[j < rank ? j : 0];
      g[i] = gain[j < rank ? j : 0];
    }
  };
  auto store = [&](int c0, float inv) {
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const int j = c0 + i * 64 + lane;
      if (j < ldc) stf(dst + j, j < rank ? ldf(&x[i]) * inv * ldf(&g[i]) : 0.0f);
    }
  };
  for (int c0 = 0; c0 < rank; c0 += 64 * N) {
    load(c0);
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const float f = c0 + i * 64 + lane < rank ? ldf(&x[i]) : 0.0f;
      ss = fmaf(f, f, ss);
    }
  }
  ss = wave_sum(ss);
  const float inv = rsq_f(ss / (float)rank + eps);
  for (int c0 = 0; c0 < ldc; c0 += 64 * N) {
    if (rank > 64 * N) load(c0);
    store(c0, inv);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void k_latent_update(const T* __restrict__ c, int64_t ld, const T* __restrict__ gain,
                                                       const int32_t* __restrict__ pos, T* __restrict__ cache, int rows,
                                                       int S, int rank, int ldc, int Smax, float eps, int32_t* err) {
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (row < rows) latent_row(c, ld, gain, pos, cache, row, S, rank, ldc, Smax, eps, err);
}

// eight consecutive values; the pointer is 16-byte aligned
__device__ __forceinline__ void ld8(const u16* p, float* f) { unpack8(ld16(p), f); }
__device__ __forceinline__ void ld8(const float* p, float* f) {
  const float4 x = *reinterpret_cast<const float4*>(p), y = *reinterpret_cast<const float4*>(p + 4);
  f[0] = x.x; f[1] = x.y; f[2] = x.z; f[3] = x.w; f[4] = y.x; f[5] = y.y; f[6] = y.z; f[7] = y.w;
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
  int S, H, share, dk, dv, window, n_keys, windowed_rows, Smax;   // share: query heads per k / v head
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
  const TK* kb = reinterpret_cast<const TK*>(a.k) + b * a.kb + h / a.share * a.kh;
  const TK* vb = reinterpret_cast<const TK*>(a.v) + b * a.vb + h / a.share * a.vh;
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

// ---- q through W_uk: q'[row, h, :] = W_uk[h]^T q[row, h, :], 16 rows and 128 latent columns of a head per workgroup, the
// head's dk rows of W_uk shared out among its four waves.  fp32 products (v_mfma_f32_16x16x4_f32) on W_uk as it lies: a lane
// reads eight consecutive columns of one row of W_uk, and column j of everybody's eight is one 16 x 16 product.  Workgroup
// h = H: the new latents, normed, into the cache (a wave per row).  The result goes out in fp32, or multiplied by `mul`
// and in bf16 (as k does where it is expanded).
struct Absorb {
  const void *q, *uk;
  int64_t ldq;
  float* out;
  u16* out_bf;
  float mul;
  int H, dk, ldr, rows, S;
  const void *c, *gain;      // latents to be cached, NULL: they already are
  int64_t ldc;
  const int32_t* pos;
  void* cache;
  int rank, Smax;
  float eps;
  int32_t* err;
};

constexpr int AW = 4;        // waves of the two projections' workgroups

template <typename T>
__global__ __launch_bounds__(64 * AW) void k_latent_absorb(const Absorb a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g4 = lane >> 4, l16 = lane & 15;
  const int row0 = blockIdx.y * 16, col0 = blockIdx.z * 128;
  if (h == a.H) {
    for (int r = blockIdx.z * AW + wave; r < 16 && row0 + r < a.rows; r += gridDim.z * AW)
      latent_row(reinterpret_cast<const T*>(a.c), a.ldc, reinterpret_cast<const T*>(a.gain), a.pos,
                 reinterpret_cast<T*>(a.cache), row0 + r, a.S, a.rank, a.ldr, a.Smax, a.eps, a.err);
    return;
  }
  const int per = ((a.dk + 4 * AW - 1) / (4 * AW)) * 4;    // rows of W_uk per wave
  float* part = sm;                                        // [AW - 1][8][4][64]
  const T* q = reinterpret_cast<const T*>(a.q) + (int64_t)min(row0 + l16, a.rows - 1) * a.ldq + h * a.dk;
  const int c = min(col0 + 8 * l16, a.ldr - 8);            // (lanes beyond the row read its last columns, for nobody)
  const T* w = reinterpret_cast<const T*>(a.uk) + (int64_t)h * a.dk * a.ldr + c;
  f32x4_t acc[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) acc[j] = f32x4_t{0, 0, 0, 0};
  constexpr int U = 4;   // steps whose loads are in flight together
  for (int d0 = 0; d0 < per; d0 += 4 * U) {
    float f[U][8], x[U];
    T xr[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int d = min(wave * per + d0 + 4 * u + g4, a.dk - 1);
      ld8(w + (int64_t)d * a.ldr, f[u]);
      xr[u] = q[d];
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      x[u] = d0 + 4 * u < per && wave * per + d0 + 4 * u + g4 < a.dk ? ldf(&xr[u]) : 0.0f;
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(f[u][j], x[u], acc[j], 0, 0, 0);
  }
  if (wave > 0) {
#pragma unroll
    for (int j = 0; j < 8; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) part[(((wave - 1) * 8 + j) * 4 + i) * 64 + lane] = acc[j][i];
  }
  __syncthreads();
  if (wave > 0) return;
#pragma unroll
  for (int v = 0; v < AW - 1; ++v)
#pragma unroll
    for (int j = 0; j < 8; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[j][i] += part[((v * 8 + j) * 4 + i) * 64 + lane];
  // register i of product j: column col0 + 8 (4 g4 + i) + j of row row0 + l16
  if (row0 + l16 >= a.rows) return;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int cc = col0 + 8 * (4 * g4 + i);
    if (cc >= a.ldr) continue;
    const int64_t at = ((int64_t)(row0 + l16) * a.H + h) * a.ldr + cc;
    float f[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) f[j] = acc[j][i];
    if (a.out) {
      st4(a.out + at, f);
      st4(a.out + at + 4, f + 4);
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) f[j] *= a.mul;
      st16(a.out_bf + at, pack8(f));
    }
  }
}

// ---- scores and sums on the latents, on the matrix cores.  One workgroup: one query row, 32 heads, a range of its
// keys, 64 at a time.  The tile of latents lies in LDS twice: by key (operand of the scores) and by column (operand of
// the weighted sums).  The fp32 softmax weights enter the bf16 products as hi + lo, which keeps them to about 2^-17.  The eight waves: (key quarter, head half) for the scores, an eighth of the latent columns for the sums.
struct Partial {
  const u16* q;              // q' [rows, H, ldr], in base-2 exponents
  const u16* cache;
  const int32_t* pos;
  float *o, *ml;             // [rows, H, nsplit, ldr], [rows, H, nsplit, 2]
  int S, H, ldr, window, Smax, nsplit;
};

constexpr int KT = 64;       // keys per tile

template <int R>
__global__ __launch_bounds__(512) void k_latent_partial(const Partial a) {
  constexpr int KS = R / 32, CROW = R + 8, VROW = KT + 8, RT = R >= 128 ? R / 128 : 1, ITEMS = R >= 128 ? R / 128 : 1;
  constexpr int SL = R >= 128 ? 16 : R / 8, PB = 64 / SL;   // a wave stages SL column slices of PB key pairs at once
  extern __shared__ __attribute__((aligned(16))) u16 su[];
  u16* Cs = su;                           // [KT][CROW]
  u16* Vt = Cs + KT * CROW;               // [R][VROW], groups of 8 keys permuted (see vgroup)
  u16* Ph = Vt + R * VROW;                // [32 heads][VROW] weights, hi and lo
  u16* Pl = Ph + 32 * VROW;
  float* mx = reinterpret_cast<float*>(Pl + 32 * VROW);   // [4][32] tile maxima of the key quarters
  float* corr = mx + 128;                 // [32]
  float* ls = corr + 32;                  // [4][32]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g4 = lane >> 4, l16 = lane & 15;
  const int sp = blockIdx.x, hb = blockIdx.y * 32, row = blockIdx.z;
  const int b = row / a.S, s = row - b * a.S;
  const int kq = wave & 3, hg = wave >> 2;
  // ---- q' of the wave's 16 heads (asked for before the position is known)
  u32x4_t qh[KS];
  {
    const int head = hb + hg * 16 + l16;
    const int64_t at = ((int64_t)row * a.H + head) * a.ldr;
#pragma unroll
    for (int j = 0; j < KS; ++j) {
      const int c = 32 * j + 8 * g4;
      qh[j] = u32x4_t{0, 0, 0, 0};
      if (head < a.H && c < a.ldr) qh[j] = *reinterpret_cast<const u32x4_t*>(a.q + at + c);
    }
  }
  const int p = min(a.pos[s], a.Smax - 1);
  const int lo = max(0, p - a.window + 1), n = p - lo + 1;
  const int per = ((n + a.nsplit - 1) / a.nsplit + KT - 1) / KT * KT;
  const int k0 = lo + sp * per, k1 = min(p + 1, k0 + per);
  const int nh = min(32, a.H - hb);
  float* mlp = a.ml + (((int64_t)row * a.H + hb) * a.nsplit + sp) * 2;
  if (k0 >= k1) {
    if (tid < nh) {
      mlp[(int64_t)tid * a.nsplit * 2] = -INFINITY;
      mlp[(int64_t)tid * a.nsplit * 2 + 1] = 0.0f;
    }
    return;
  }
  // Staging: an item is eight columns of two neighbouring keys, stored by column as dwords of two keys.  Column slices
  // that a wave writes together would meet in two LDS banks (their rows lie 8 * 36 dwords apart): the groups of eight
  // keys of a row are permuted by its slice, which spreads them over all banks and leaves a group whole for the reader.
  const rsrc_t res = buffer_of(a.cache + (int64_t)b * a.Smax * a.ldr, a.Smax * a.ldr * 2);
  u32x4_t st[ITEMS][2];
  auto slot = [&](int i, int& kp, int& c) {
    const int blk = i * 8 + wave;                   // PB key pairs x SL slices
    constexpr int NP = (KT / 2) / PB;
    kp = (blk % NP) * PB + lane / SL;
    c = ((blk / NP) * SL + lane % SL) * 8;
  };
  auto stage_load = [&](int t0) {
#pragma unroll
    for (int i = 0; i < ITEMS; ++i) {
      int kp, c;
      slot(i, kp, c);
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int key = t0 + 2 * kp + e;
        st[i][e] = __builtin_amdgcn_raw_buffer_load_b128(res, (c < a.ldr && key < k1) ? (key * a.ldr + c) * 2 : NOWHERE, 0, 0);
      }
    }
  };
  auto vgroup = [](int group, int r) { return group ^ ((r >> 4) & 7); };
  stage_load(k0);
  f32x4_t o[2][RT];
#pragma unroll
  for (int g = 0; g < 2; ++g)
#pragma unroll
    for (int t = 0; t < RT; ++t) o[g][t] = f32x4_t{0, 0, 0, 0};
  float m[4] = {-INFINITY, -INFINITY, -INFINITY, -INFINITY}, l[4] = {0, 0, 0, 0};
  u32* vt32 = reinterpret_cast<u32*>(Vt);
  const int cw = wave * 16 * RT;          // this wave's first column in the sums
  for (int t0 = k0; t0 < k1; t0 += KT) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < ITEMS; ++i) {
      int kp, c;
      slot(i, kp, c);
      if (c < R) {
#pragma unroll
        for (int e = 0; e < 2; ++e) *reinterpret_cast<u32x4_t*>(&Cs[(2 * kp + e) * CROW + c]) = st[i][e];
        const int at = vgroup(kp >> 2, c) * 4 + (kp & 3);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          vt32[(c + 2 * j) * (VROW / 2) + at] = (st[i][0][j] & 0xffffu) | (st[i][1][j] << 16);
          vt32[(c + 2 * j + 1) * (VROW / 2) + at] = (st[i][0][j] >> 16) | (st[i][1][j] & 0xffff0000u);
        }
      }
    }
    __syncthreads();
    if (t0 + KT < k1) stage_load(t0 + KT);
    // ---- scores: rows are heads, columns keys
    f32x4_t sa = {0, 0, 0, 0}, sb = {0, 0, 0, 0};
#pragma unroll
    for (int j = 0; j < KS; ++j) {
      const u32x4_t kc = *reinterpret_cast<const u32x4_t*>(&Cs[(kq * 16 + l16) * CROW + 32 * j + 8 * g4]);
      f32x4_t& acc = j & 1 ? sb : sa;
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, qh[j]), __builtin_bit_cast(bf16x8_t, kc), acc, 0, 0, 0);
    }
    sa += sb;
    const bool seen = t0 + kq * 16 + l16 < k1;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      sa[i] = seen ? sa[i] : -INFINITY;
      const float t = row16_max(sa[i]);
      if (l16 == 0) mx[kq * 32 + hg * 16 + 4 * g4 + i] = t;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int hh = hg * 16 + 4 * g4 + i;
      const float mt = fmaxf(fmaxf(mx[hh], mx[32 + hh]), fmaxf(mx[64 + hh], mx[96 + hh]));
      const float mn = fmaxf(m[i], mt);   // finite: the tile's first key is seen
      const float cr = exp2_f(m[i] - mn), w = exp2_f(sa[i] - mn);
      m[i] = mn;
      l[i] = l[i] * cr + w;
      Ph[hh * VROW + kq * 16 + l16] = f_to_bf(w);
      Pl[hh * VROW + kq * 16 + l16] = f_to_bf(w - round_bf(w));
      if (kq == 0 && l16 == 0) corr[hh] = cr;
    }
    __syncthreads();
    // ---- sums: this wave's columns, keys 32 at a time
    if (cw < R) {
      bf16x8_t ph[2][2], pl[2][2];
#pragma unroll
      for (int g = 0; g < 2; ++g)
#pragma unroll
        for (int k = 0; k < 2; ++k) {
          ph[g][k] = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(&Ph[(16 * g + l16) * VROW + 32 * k + 8 * g4]));
          pl[g][k] = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(&Pl[(16 * g + l16) * VROW + 32 * k + 8 * g4]));
        }
      f32x4_t cv[2];
#pragma unroll
      for (int g = 0; g < 2; ++g) {
        const float4 c = *reinterpret_cast<const float4*>(&corr[16 * g + 4 * g4]);
        cv[g] = f32x4_t{c.x, c.y, c.z, c.w};
      }
#pragma unroll
      for (int t = 0; t < RT; ++t) {
        const int r = cw + 16 * t + l16;
        o[0][t] *= cv[0];
        o[1][t] *= cv[1];
#pragma unroll
        for (int k = 0; k < 2; ++k) {
          const bf16x8_t vt = __builtin_bit_cast(bf16x8_t, *reinterpret_cast<const u32x4_t*>(&Vt[r * VROW + 8 * vgroup(4 * k + g4, r)]));
          o[0][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ph[0][k], vt, o[0][t], 0, 0, 0);
          o[1][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ph[1][k], vt, o[1][t], 0, 0, 0);
          o[0][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl[0][k], vt, o[0][t], 0, 0, 0);
          o[1][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl[1][k], vt, o[1][t], 0, 0, 0);
        }
      }
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float t = row16_sum(l[i]);
    const int hh = hg * 16 + 4 * g4 + i;
    if (l16 == 0) {
      ls[kq * 32 + hh] = t;
      if (kq == 0) mx[hh] = m[i];   // (nobody reads the last tile's maxima any more: a barrier lies between)
    }
  }
  __syncthreads();
  if (tid < nh) {
    mlp[(int64_t)tid * a.nsplit * 2] = mx[tid];
    mlp[(int64_t)tid * a.nsplit * 2 + 1] = (ls[tid] + ls[32 + tid]) + (ls[64 + tid] + ls[96 + tid]);
  }
  if (cw >= R) return;
#pragma unroll
  for (int g = 0; g < 2; ++g)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int hh = g * 16 + 4 * g4 + i;
      if (hh < nh) {
        float* op = a.o + (((int64_t)row * a.H + hb + hh) * a.nsplit + sp) * a.ldr;
#pragma unroll
        for (int t = 0; t < RT; ++t) {
          const int c = cw + 16 * t + l16;
          if (c < a.ldr) op[c] = o[g][t][i];
        }
      }
    }
}

// ---- the ranges' results merged, then through W_uv: y[row, h dv + e] = W_uv[h dv + e, :] . o[row, h, :], UR rows and 64
// value dimensions of a head per workgroup.  Eight waves: (16 value dimensions, half of the latent columns).  bf16: the
// fp32 o enters the products as hi + lo; fp32: fp32 products.
constexpr int UR = 4, UT = 512;

template <typename T, int SB>
__global__ __launch_bounds__(UT) void k_latent_up(const float* __restrict__ o, const float* __restrict__ ml,
                                                  const T* __restrict__ uv, T* __restrict__ y, int64_t ldy, int H, int dv,
                                                  int ldr, int nsplit, int rows) {
  constexpr bool BF = sizeof(T) == 2;
  extern __shared__ __attribute__((aligned(16))) float os[];   // fp32: [16][orow]; bf16: hi [16][orow], lo [16][orow]
  __shared__ float ws[UR][64];
  __shared__ float part[4][64][4];
  const int kp = (ldr + 63) / 64 * 64, orow = kp + 8;
  u16 *oh = reinterpret_cast<u16*>(os), *ol = oh + 16 * orow;
  const int h = blockIdx.x, row0 = blockIdx.y * UR, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int g4 = lane >> 4, l16 = lane & 15;
  const int nr = min(UR, rows - row0);
  // this wave's rows of W_uv, 32 columns a step: lane (g4, l16) has eight columns of row l16.  The first steps' loads are
  // out before the merge begins.
  const int e0 = blockIdx.z * 64 + (wave & 3) * 16, cb = (wave >> 2) * (kp / 2), ce = cb + kp / 2;
  constexpr int U = 8;
  const T* w = uv + ((int64_t)h * dv + min(e0 + l16, dv - 1)) * ldr;
  T wx[U][8];
  auto load = [&](int c0) {
#pragma unroll
    for (int u = 0; u < U; ++u)
      __builtin_memcpy(wx[u], __builtin_assume_aligned(w + min(c0 + 32 * u + 8 * g4, ldr - 8), 16), sizeof(wx[u]));
  };
  load(cb);
  // ---- an item is four columns of a row; its ranges' values, SB at a time, do not wait for the ranges' weights.  A range
  // beyond the last repeats the last one's place with weight 0.
  const int q4 = kp / 4, items = UR * q4;
  const int ns = ml ? nsplit : 1;
  float4 x[SB];
  auto fetch = [&](int i, int s0) {
    const int r = i / q4, c = (i - r * q4) * 4;
    const float* p = o + ((int64_t)(row0 + min(r, nr - 1)) * H + h) * ns * ldr + min(c, ldr - 4);
#pragma unroll
    for (int s = 0; s < SB; ++s)
      if (s0 + s < ns) x[s] = *reinterpret_cast<const float4*>(p + (int64_t)(s0 + s) * ldr);
  };
  fetch(min(tid, items - 1), 0);
  if (wave < UR) {
    // weight of every range: 2^(m - M) / sum of 2^(m - M) l
    const float* p = ml + ((int64_t)(row0 + min(wave, nr - 1)) * H + h) * nsplit * 2;
    float m = lane == 0 ? 0.0f : -INFINITY, l = 1.0f;
    if (ml) {
      m = lane < nsplit ? p[2 * lane] : -INFINITY;
      l = lane < nsplit ? p[2 * lane + 1] : 0.0f;
    }
    const float f = exp2_f(m - wave_max(m));
    ws[wave][lane] = f / wave_sum(f * l);
  }
  // (rows of the products that are nobody's)
  for (int i = tid; i < (16 - UR) * orow; i += UT) {
    if constexpr (BF) oh[UR * orow + i] = ol[UR * orow + i] = 0;
    else os[UR * orow + i] = 0.0f;
  }
  __syncthreads();
  for (int i = tid; i < items; i += UT) {
    const int r = i / q4, c = (i - r * q4) * 4;
    float t[4] = {0, 0, 0, 0};
    for (int s0 = 0; s0 < ns; s0 += SB) {
      if (i != tid || s0 > 0) fetch(i, s0);
#pragma unroll
      for (int s = 0; s < SB; ++s)
        if (s0 + s < ns) {
          const float f = ws[r][s0 + s];   // 0: nothing was written there
          t[0] += f > 0.0f ? f * x[s].x : 0.0f;
          t[1] += f > 0.0f ? f * x[s].y : 0.0f;
          t[2] += f > 0.0f ? f * x[s].z : 0.0f;
          t[3] += f > 0.0f ? f * x[s].w : 0.0f;
        }
    }
    const bool ok = r < nr && c < ldr;
#pragma unroll
    for (int j = 0; j < 4; ++j) t[j] = ok ? t[j] : 0.0f;
    if constexpr (BF) {
      st4(&oh[r * orow + c], t);
#pragma unroll
      for (int j = 0; j < 4; ++j) t[j] -= round_bf(t[j]);
      st4(&ol[r * orow + c], t);
    } else {
      st4(&os[r * orow + c], t);
    }
  }
  __syncthreads();
  f32x4_t acc[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}};
  for (int c0 = cb; c0 < ce; c0 += 32 * U) {
    if (c0 > cb) load(c0);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = c0 + 32 * u + 8 * g4;
      if (c0 + 32 * u >= ce) break;         // uniform
      if constexpr (BF) {
        bf16x8_t a;
        __builtin_memcpy(&a, wx[u], sizeof(a));
        const u32x4_t zh = *reinterpret_cast<const u32x4_t*>(&oh[l16 * orow + c]);
        const u32x4_t zl = *reinterpret_cast<const u32x4_t*>(&ol[l16 * orow + c]);
        acc[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, __builtin_bit_cast(bf16x8_t, zh), acc[0], 0, 0, 0);
        acc[1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, __builtin_bit_cast(bf16x8_t, zl), acc[1], 0, 0, 0);
      } else {
        float z[8];
        ld8(&os[l16 * orow + c], z);
#pragma unroll
        for (int i = 0; i < 8; ++i)
          acc[i & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(ldf(&wx[u][i]), z[i], acc[i & 1], 0, 0, 0);
      }
    }
  }
  acc[0] += acc[1];
  if (wave >= 4) {
#pragma unroll
    for (int i = 0; i < 4; ++i) part[wave & 3][lane][i] = acc[0][i];
  }
  __syncthreads();
  if (wave >= 4 || l16 >= nr) return;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int e = e0 + 4 * g4 + i;
    if (e < dv) stf(y + (int64_t)(row0 + l16) * ldy + h * dv + e, acc[0][i] + part[wave][lane][i]);
  }
}

template <typename TQ, typename TK, typename TO>
int launch_window(const WinAttn& a, int B, hipStream_t s) {
  const size_t lds = sizeof(float) * (((a.dk + 3) & ~3) + 64);
  k_window_attention<TQ, TK, TO><<<dim3(a.H, a.S, B), dim3(64), lds, s>>>(a);
  return lr_launch_status();
}

// Key ranges per query row of the matrix-core kernel: about a workgroup per CU, no range shorter than a tile.
int splits(int rows, int H, int window, int Smax) {
  const int keys = window < Smax ? window : Smax;
  const int64_t wgs = (int64_t)rows * ((H + 31) / 32);
  int64_t n = (256 + wgs - 1) / wgs;
  const int most = (keys + KT - 1) / KT;
  if (n > most) n = most;
  return n > 64 ? 64 : (int)n;
}

template <int R>
int launch_partial(const Partial& a, int rows, hipStream_t s) {
  const size_t lds = sizeof(u16) * ((size_t)KT * (R + 8) + (R + 2 * 32) * (KT + 8)) + sizeof(float) * 288;
  static std::atomic<unsigned long long> raised{0};
  if (!lr_raise_lds_limit(reinterpret_cast<const void*>(&k_latent_partial<R>), lds, raised)) return LR_E_LAUNCH;
  k_latent_partial<R><<<dim3(a.nsplit, (a.H + 31) / 32, rows), dim3(512), lds, s>>>(a);
  return lr_launch_status();
}

template <typename T>
int absorb(const Absorb& a, hipStream_t s) {
  const size_t lds = sizeof(float) * (AW - 1) * 8 * 4 * 64;
  k_latent_absorb<T><<<dim3(a.H + (a.c ? 1 : 0), (a.rows + 15) / 16, (a.ldr + 127) / 128), dim3(64 * AW), lds, s>>>(a);
  return lr_launch_status();
}

template <typename T, int SB>
int up_as(const float* o, const float* ml, const lr_latent_attention_t* d, int rows, int nsplit, hipStream_t s) {
  const size_t lds = (size_t)16 * ((d->ldr + 63) / 64 * 64 + 8) * sizeof(float);   // (hi and lo, or fp32)
  static std::atomic<unsigned long long> raised{0};
  if (!lr_raise_lds_limit(reinterpret_cast<const void*>(&k_latent_up<T, SB>), lds, raised)) return LR_E_LAUNCH;
  k_latent_up<T, SB><<<dim3(d->H, (rows + UR - 1) / UR, (d->dv + 63) / 64), dim3(UT), lds, s>>>(
      o, ml, (const T*)d->uv, (T*)d->y, d->ldy, d->H, d->dv, d->ldr, nsplit, rows);
  return lr_launch_status();
}

// (the registers of eight ranges' values instead of sixteen's leave room for a second workgroup on a CU)
template <typename T>
int up(const float* o, const float* ml, const lr_latent_attention_t* d, int rows, int nsplit, hipStream_t s) {
  return nsplit <= 8 ? up_as<T, 8>(o, ml, d, rows, nsplit, s) : up_as<T, 16>(o, ml, d, rows, nsplit, s);
}

template <typename T>
int latent_attention(const lr_latent_attention_t* d, hipStream_t s) {
  float* qa = reinterpret_cast<float*>(d->scratch);
  const int rows = d->B * d->S;
  float* ol = qa + (size_t)rows * d->H * d->ldr;
  // bf16: q' scaled to base-2 exponents, for the matrix-core kernel
  const bool split = d->dtype == LR_BF16 && d->ldr <= 512 && d->scale > 0.0f && (int64_t)d->Smax * d->ldr * 2 < 0x7fffffff;
  u16* qb = reinterpret_cast<u16*>(qa);
  Absorb ab = {d->q, d->uk, d->ldq, split ? nullptr : qa, qb, d->scale * LOG2E, d->H, d->dk, d->ldr, rows, d->S,
               d->latent, d->norm, d->ldl, d->pos, d->cache, d->rank, d->Smax, d->eps, d->err};
  int rc = absorb<T>(ab, s);
  if (rc != LR_OK) return rc;
  float* ml = nullptr;
  int ns = 1;
  if (split) {
    ns = splits(rows, d->H, d->window, d->Smax);
    ml = ol + (size_t)rows * d->H * ns * d->ldr;
    const Partial p = {qb, (const u16*)d->cache, d->pos, ol, ml, d->S, d->H, d->ldr, d->window, d->Smax, ns};
    rc = d->ldr <= 64 ? launch_partial<64>(p, rows, s) : d->ldr <= 128 ? launch_partial<128>(p, rows, s)
         : d->ldr <= 256 ? launch_partial<256>(p, rows, s) : launch_partial<512>(p, rows, s);
  } else {
    WinAttn a = {};
    a.q = qa; a.ldq = (int64_t)d->H * d->ldr; a.hq = d->ldr;
    a.k = a.v = d->cache;
    a.kb = a.vb = (int64_t)d->Smax * d->ldr; a.kr = a.vr = d->ldr; a.kh = a.vh = 0;
    a.y = ol; a.ldy = a.ldq; a.hy = d->ldr; a.pos = d->pos;
    a.S = d->S; a.H = d->H; a.share = 1; a.dk = a.dv = d->ldr; a.window = d->window; a.n_keys = d->Smax; a.Smax = d->Smax;
    a.scale = d->scale;
    rc = launch_window<float, T, float>(a, d->B, s);
  }
  if (rc != LR_OK) return rc;
  return up<T>(ol, ml, d, rows, ns, s);
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
      d->n_keys > d->Smax || d->kv_heads < 0)
    return LR_E_SHAPE;
  const int G = d->kv_heads > 0 ? d->kv_heads : d->H;
  if (d->H % G) return LR_E_SHAPE;
  if (d->ldq < (int64_t)d->H * d->dk || d->ldy < (int64_t)d->H * d->dv || d->ldk < (int64_t)G * d->dk ||
      d->ldk < (int64_t)G * d->dv)
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
  a.S = d->S; a.H = d->H; a.share = d->H / G; a.dk = d->dk; a.dv = d->dv; a.window = d->window; a.n_keys = d->n_keys; a.windowed_rows = 1;
  a.Smax = d->Smax; a.scale = d->scale;
  hipStream_t s = (hipStream_t)stream;
  if (d->dtype == LR_BF16) return launch_window<u16, u16, u16>(a, d->B, s);
  if (d->dtype == LR_F32) return launch_window<float, float, float>(a, d->B, s);
  return LR_E_UNSUPPORTED;
}

extern "C" size_t lr_latent_attention_scratch_bytes(int B, int S, int H, int ldr, int window, int Smax) {
  if (B <= 0 || S <= 0 || H <= 0 || ldr <= 0 || window <= 0 || Smax <= 0) return 0;
  const size_t ns = splits(B * S, H, window, Smax);
  return (size_t)B * S * H * (ldr + ns * (ldr + 2)) * sizeof(float);
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
  if (d->scratch_bytes < lr_latent_attention_scratch_bytes(d->B, d->S, d->H, d->ldr, d->window, d->Smax)) return LR_E_SHAPE;
  if (d->latent) {
    LR_REQUIRE_PTR(d->norm);
    if (d->rank <= 0 || d->rank > d->ldr || d->ldl < d->rank) return LR_E_SHAPE;
  }
  if (d->ldr % 8) return LR_E_ALIGN;
  if (d->ldr > 1024 || (int64_t)d->B * d->S > 65535 || d->dk > 2048) return LR_E_UNSUPPORTED;
  if (d->dtype == LR_BF16) return latent_attention<u16>(d, (hipStream_t)stream);
  if (d->dtype == LR_F32) return latent_attention<float>(d, (hipStream_t)stream);
  return LR_E_UNSUPPORTED;
}
