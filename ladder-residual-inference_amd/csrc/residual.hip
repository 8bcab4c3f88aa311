// Models that keep their residual stream in fp32: embedding, residual update + RMS norm, capped logits; and the plain
// fp32 linear and SwiGLU for running such a model in fp32 throughout.
#include "mixer_common.h"

namespace {

// x[t, :] = table[idx[t], :] * scale in fp32, and the same in the compute type (the first mixer's input)
template <typename T>
__global__ __launch_bounds__(256) void k_embed_residual(const T* __restrict__ table, const void* __restrict__ idx,
                                                        int idx_is_i64, float* __restrict__ x, T* __restrict__ xc,
                                                        int dim, int vocab, float scale) {
  const int64_t t = blockIdx.x;
  const int64_t id = idx_is_i64 ? reinterpret_cast<const int64_t*>(idx)[t]
                                : (int64_t) reinterpret_cast<const int32_t*>(idx)[t];
  const bool ok = id >= 0 && id < vocab;
  const T* src = table + (ok ? id : 0) * (int64_t)dim;
  for (int c = threadIdx.x * 4; c < dim; c += 256 * 4) {
    Quad<T> r;
    r.load(src + c);
    float f[4];
    r.get(f);
#pragma unroll
    for (int j = 0; j < 4; ++j) f[j] = ok ? f[j] * scale : 0.0f;
    st4(x + t * dim + c, f);
    if (xc) st4(xc + t * dim + c, f);
  }
}

// r = alpha x + d;  out = r / sqrt(mean(r^2) + eps) * (offset + gain), in fp32 and / or in the compute type.  The mean is
// over the first `width` columns (the rest is padding: zero in, zero out).
constexpr int RN_MAXIT = 16;  // 256 lanes x 4 columns x 16
template <typename T, int RN_IT>
__global__ __launch_bounds__(256) void k_residual_norm(const float* x, float alpha, const T* __restrict__ d,
                                                       const T* __restrict__ gain, float offset, float* xo,
                                                       T* __restrict__ xc, int dim, int width, float eps) {
  __shared__ float red[4];
  const int tid = threadIdx.x;
  const int64_t base = (int64_t)blockIdx.x * dim;
  float4 qx[RN_IT];
  Quad<T> qd[RN_IT], qg[RN_IT];
#pragma unroll
  for (int i = 0; i < RN_IT; ++i) {
    const int c0 = (tid + i * 256) * 4, c = c0 < dim ? c0 : 0;
    qx[i] = *reinterpret_cast<const float4*>(x + base + c);
    if (d) qd[i].load(d + base + c);
    qg[i].load(gain + c);
  }
  float ss = 0.0f;
#pragma unroll
  for (int i = 0; i < RN_IT; ++i) {
    const int c = (tid + i * 256) * 4;
    float f[4] = {0, 0, 0, 0};
    if (d) qd[i].get(f);
    qx[i].x = fmaf(alpha, qx[i].x, f[0]);
    qx[i].y = fmaf(alpha, qx[i].y, f[1]);
    qx[i].z = fmaf(alpha, qx[i].z, f[2]);
    qx[i].w = fmaf(alpha, qx[i].w, f[3]);
    if (c < dim) ss += (qx[i].x * qx[i].x + qx[i].y * qx[i].y) + (qx[i].z * qx[i].z + qx[i].w * qx[i].w);
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  const float inv = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)width + eps);
#pragma unroll
  for (int i = 0; i < RN_IT; ++i) {
    const int c = (tid + i * 256) * 4;
    if (c < dim) {
      float g[4];
      qg[i].get(g);
      const float o[4] = {qx[i].x * inv * (offset + g[0]), qx[i].y * inv * (offset + g[1]),
                          qx[i].z * inv * (offset + g[2]), qx[i].w * inv * (offset + g[3])};
      if (xo) st4(xo + base + c, o);
      if (xc) st4(xc + base + c, o);
    }
  }
}

// r = x + d + sum over a token's slots of weight * out (the experts of a mixture);  x_out = r and
// x_compute = tanh(alpha r) gain + bias: a norm without statistics, so a row is cut into as many workgroups as it fills.
template <typename T>
__global__ __launch_bounds__(256) void k_residual_tanh(const float* x, const T* __restrict__ d, const T* __restrict__ eo,
                                                       const float* __restrict__ ew, int top, const T* __restrict__ alpha,
                                                       const T* __restrict__ gain, const T* __restrict__ bias, float* xo,
                                                       T* __restrict__ xc, int dim) {
  const int64_t row = blockIdx.x;
  const int c = (blockIdx.y * 256 + threadIdx.x) * 4;
  if (c >= dim) return;
  const int64_t at = row * dim + c;
  const float4 q = *reinterpret_cast<const float4*>(x + at);
  float r[4] = {q.x, q.y, q.z, q.w};
  if (d) {
    Quad<T> t;
    t.load(d + at);
    float f[4];
    t.get(f);
#pragma unroll
    for (int j = 0; j < 4; ++j) r[j] += f[j];
  }
  if (eo) {
    float s[4] = {0, 0, 0, 0};
#pragma unroll 4
    for (int k = 0; k < top; ++k) {
      const float w = ew[row * top + k];
      Quad<T> t;
      t.load(eo + (row * top + k) * dim + c);
      float f[4];
      t.get(f);
#pragma unroll
      for (int j = 0; j < 4; ++j) s[j] = fmaf(w, f[j], s[j]);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) r[j] += s[j];
  }
  if (xo) st4(xo + at, r);
  if (xc) {
    Quad<T> tg, tb;
    tg.load(gain + c);
    tb.load(bias + c);
    float g[4], b[4];
    tg.get(g);
    tb.get(b);
    const float al = ldf(alpha);
#pragma unroll
    for (int j = 0; j < 4; ++j) r[j] = fmaf(tanhf(al * r[j]), g[j], b[j]);
    st4(xc + at, r);
  }
}

// logits <- cap tanh(scale logits / cap), in place (cap <= 0: the scale alone)
template <typename T>
__global__ __launch_bounds__(256) void k_logit_cap(T* l, int64_t ld, int V, float scale, float cap) {
  T* row = l + (int64_t)blockIdx.x * ld;
  for (int c = blockIdx.y * 256 + threadIdx.x; c < V; c += gridDim.y * 256) {
    const float z = ldf(row + c) * scale;
    stf(row + c, cap > 0.0f ? cap * tanhf(z / cap) : z);
  }
}

// y = x w^T in fp32: 64 x 64 tiles, four waves of 32 x 32, v_mfma_f32_16x16x4_f32; any M, N, K.  GROUP: the rows of a tile
// are entries of a list, tile (matrix, first entry, entries) as a device table says: input row entry / xdiv, output row
// entry, weights of one of several matrices.
constexpr int FT = 64, FK = 16, FL = FK + 4;
template <bool GROUP>
__global__ __launch_bounds__(256) void k_linear_f32(const float* __restrict__ x, int64_t ldx, const float* __restrict__ w,
                                                    float* __restrict__ y, int64_t ldy, int M, int N, int K,
                                                    const int32_t* __restrict__ tiles, const int32_t* __restrict__ ntiles,
                                                    const int32_t* __restrict__ entries, int xdiv) {
  __shared__ __attribute__((aligned(16))) float xs[FT * FL], ws[FT * FL];
  __shared__ int32_t rows[FT];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g4 = lane >> 4, l16 = lane & 15;
  if constexpr (GROUP) {
    if ((int)blockIdx.y >= ntiles[0]) return;
    const int32_t* tile = tiles + 3 * blockIdx.y;
    w += (int64_t)tile[0] * N * K;
    M = tile[2];
    if (tid < FT) rows[tid] = entries[tile[1] + (tid < M ? tid : 0)];
    __syncthreads();
  }
  const int m0 = GROUP ? 0 : blockIdx.y * FT, n0 = blockIdx.x * FT, wm = (wave >> 1) * 32, wn = (wave & 1) * 32;
  f32x4_t acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = f32x4_t{0, 0, 0, 0};
  const int r = tid >> 2, c4 = (tid & 3) * 4;
  const int64_t xrow = GROUP ? rows[r] / xdiv : m0 + r;
  for (int k0 = 0; k0 < K; k0 += FK) {
    float fx[4], fw[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int kk = k0 + c4 + j;
      fx[j] = (m0 + r < M && kk < K) ? x[xrow * ldx + kk] : 0.0f;
      fw[j] = (n0 + r < N && kk < K) ? w[(int64_t)(n0 + r) * K + kk] : 0.0f;
    }
    __syncthreads();
    st4(&xs[r * FL + c4], fx);
    st4(&ws[r * FL + c4], fw);
    __syncthreads();
    float4 a[2], b[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      a[i] = *reinterpret_cast<const float4*>(&xs[(wm + 16 * i + l16) * FL + 4 * g4]);
      b[i] = *reinterpret_cast<const float4*>(&ws[(wn + 16 * i + l16) * FL + 4 * g4]);
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i].x, b[j].x, acc[i][j], 0, 0, 0);
        acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i].y, b[j].y, acc[i][j], 0, 0, 0);
        acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i].z, b[j].z, acc[i][j], 0, 0, 0);
        acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i].w, b[j].w, acc[i][j], 0, 0, 0);
      }
  }
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int m = m0 + wm + 16 * i + 4 * g4 + e, n = n0 + wn + 16 * j + l16;
        if (m < M && n < N) y[(int64_t)(GROUP ? rows[m] : m) * ldy + n] = acc[i][j][e];
      }
}

__global__ __launch_bounds__(256) void k_swiglu_f32(const float* __restrict__ h, int64_t ldh, float* __restrict__ out,
                                                    int64_t ldo, int I) {
  const float* row = h + (int64_t)blockIdx.x * ldh;
  for (int c = threadIdx.x; c < I; c += 256) out[(int64_t)blockIdx.x * ldo + c] = silu_f(row[I + c]) * row[c];
}

template <typename T>
void launch_residual_norm(const float* x, float alpha, const T* d, const T* gain, float offset, float* xo, T* xc, int rows,
                          int dim, int width, float eps, hipStream_t s) {
#define LR_RN(IT)                                                                                                    \
  if (dim <= 1024 * IT) {                                                                                            \
    k_residual_norm<T, IT><<<dim3(rows), dim3(256), 0, s>>>(x, alpha, d, gain, offset, xo, xc, dim, width, eps);      \
    return;                                                                                                          \
  }
  LR_RN(1) LR_RN(2) LR_RN(4) LR_RN(8) LR_RN(16)
#undef LR_RN
}

}  // namespace

extern "C" int lr_embed_residual(const void* table, const void* idx, int idx_is_i64, float* x, void* x_compute,
                                 int64_t n_tokens, int dim, int vocab, float scale, int dtype, lr_stream_t stream) {
  LR_REQUIRE_PTR(table);
  LR_REQUIRE_PTR(x);
  LR_OPTIONAL_PTR(x_compute);
  if (idx == nullptr) return LR_E_NULL;
  if (n_tokens <= 0 || dim <= 0 || vocab <= 0 || n_tokens > 0x7fffffff) return LR_E_SHAPE;
  if (dim % 8) return LR_E_ALIGN;
  const dim3 grid((unsigned)n_tokens), blk(256);
  if (dtype == LR_BF16)
    k_embed_residual<u16><<<grid, blk, 0, (hipStream_t)stream>>>((const u16*)table, idx, idx_is_i64, x, (u16*)x_compute,
                                                                dim, vocab, scale);
  else if (dtype == LR_F32)
    k_embed_residual<float><<<grid, blk, 0, (hipStream_t)stream>>>((const float*)table, idx, idx_is_i64, x,
                                                                  (float*)x_compute, dim, vocab, scale);
  else
    return LR_E_UNSUPPORTED;
  return lr_launch_status();
}

extern "C" int lr_residual_rmsnorm(const float* x, float alpha, const void* d, const void* gain, float gain_offset,
                                   float* x_out, void* x_compute, int rows, int dim, int width, float eps, int dtype,
                                   lr_stream_t stream) {
  LR_REQUIRE_PTR(x);
  LR_REQUIRE_PTR(gain);
  LR_OPTIONAL_PTR(d);
  LR_OPTIONAL_PTR(x_out);
  LR_OPTIONAL_PTR(x_compute);
  if (x_out == nullptr && x_compute == nullptr) return LR_E_NULL;
  if (rows <= 0 || dim <= 0 || width <= 0 || width > dim) return LR_E_SHAPE;
  if (dim % 8) return LR_E_ALIGN;
  if (dim > 1024 * RN_MAXIT) return LR_E_UNSUPPORTED;
  if (dtype == LR_BF16)
    launch_residual_norm<u16>(x, alpha, (const u16*)d, (const u16*)gain, gain_offset, x_out, (u16*)x_compute, rows, dim,
                              width, eps, (hipStream_t)stream);
  else if (dtype == LR_F32)
    launch_residual_norm<float>(x, alpha, (const float*)d, (const float*)gain, gain_offset, x_out, (float*)x_compute, rows,
                                dim, width, eps, (hipStream_t)stream);
  else
    return LR_E_UNSUPPORTED;
  return lr_launch_status();
}

extern "C" int lr_residual_tanh(const float* x, const void* d, const void* expert_out, const float* expert_weights, int top,
                                const void* alpha, const void* gain, const void* bias, float* x_out, void* x_compute, int rows,
                                int dim, int dtype, lr_stream_t stream) {
  LR_REQUIRE_PTR(x);
  LR_OPTIONAL_PTR(d);
  LR_OPTIONAL_PTR(expert_out);
  LR_OPTIONAL_PTR(x_out);
  LR_OPTIONAL_PTR(x_compute);
  if (x_out == nullptr && x_compute == nullptr) return LR_E_NULL;
  if (x_compute) {
    LR_REQUIRE_PTR(gain);
    LR_REQUIRE_PTR(bias);
    if (alpha == nullptr) return LR_E_NULL;
  }
  if (expert_out && expert_weights == nullptr) return LR_E_NULL;
  if (rows <= 0 || dim <= 0 || (expert_out && top <= 0)) return LR_E_SHAPE;
  if (dim % 8) return LR_E_ALIGN;
  if (dim > 1024 * 65535) return LR_E_UNSUPPORTED;
  const dim3 grid(rows, (dim + 1023) / 1024), blk(256);
  if (dtype == LR_BF16)
    k_residual_tanh<u16><<<grid, blk, 0, (hipStream_t)stream>>>(x, (const u16*)d, (const u16*)expert_out, expert_weights, top,
                                                               (const u16*)alpha, (const u16*)gain, (const u16*)bias, x_out,
                                                               (u16*)x_compute, dim);
  else if (dtype == LR_F32)
    k_residual_tanh<float><<<grid, blk, 0, (hipStream_t)stream>>>(x, (const float*)d, (const float*)expert_out, expert_weights, top,
                                                                 (const float*)alpha, (const float*)gain, (const float*)bias, x_out,
                                                                 (float*)x_compute, dim);
  else
    return LR_E_UNSUPPORTED;
  return lr_launch_status();
}

extern "C" int lr_logit_cap(void* logits, int64_t ldl, int rows, int V, float scale, float cap, int dtype,
                            lr_stream_t stream) {
  LR_REQUIRE_PTR(logits);
  if (rows <= 0 || V <= 0 || ldl < V) return LR_E_SHAPE;
  int gy = (V + 2047) / 2048;
  gy = gy > 64 ? 64 : gy;
  if (dtype == LR_BF16)
    k_logit_cap<u16><<<dim3(rows, gy), dim3(256), 0, (hipStream_t)stream>>>((u16*)logits, ldl, V, scale, cap);
  else if (dtype == LR_F32)
    k_logit_cap<float><<<dim3(rows, gy), dim3(256), 0, (hipStream_t)stream>>>((float*)logits, ldl, V, scale, cap);
  else
    return LR_E_UNSUPPORTED;
  return lr_launch_status();
}

extern "C" int lr_linear_f32(const float* x, int64_t ldx, const float* w, float* y, int64_t ldy, int M, int N, int K,
                             lr_stream_t stream) {
  LR_REQUIRE_PTR(x);
  LR_REQUIRE_PTR(w);
  LR_REQUIRE_PTR(y);
  if (M <= 0 || N <= 0 || K <= 0 || ldx < K || ldy < N) return LR_E_SHAPE;
  const dim3 grid((N + FT - 1) / FT, (M + FT - 1) / FT);
  if (grid.y > 65535) return LR_E_UNSUPPORTED;
  k_linear_f32<false><<<grid, dim3(256), 0, (hipStream_t)stream>>>(x, ldx, w, y, ldy, M, N, K, nullptr, nullptr, nullptr, 1);
  return lr_launch_status();
}

namespace lr_detail {
int linear_f32_grouped(const float* x, int64_t ldx, const float* w, float* y, int64_t ldy, int N, int K, const int32_t* tiles,
                       const int32_t* ntiles, const int32_t* entries, int xdiv, int max_tiles, hipStream_t s) {
  if (max_tiles > 65535) return LR_E_UNSUPPORTED;
  k_linear_f32<true><<<dim3((N + FT - 1) / FT, max_tiles), dim3(256), 0, s>>>(x, ldx, w, y, ldy, FT, N, K, tiles, ntiles, entries, xdiv);
  return lr_launch_status();
}
int linear_f32_grouped_rows() { return FT; }
}  // namespace lr_detail

extern "C" int lr_swiglu_f32(const float* h, int64_t ldh, float* out, int64_t ldo, int rows, int I, lr_stream_t stream) {
  LR_REQUIRE_PTR(h);
  LR_REQUIRE_PTR(out);
  if (rows <= 0 || I <= 0 || ldh < 2 * (int64_t)I || ldo < I) return LR_E_SHAPE;
  k_swiglu_f32<<<dim3(rows), dim3(256), 0, (hipStream_t)stream>>>(h, ldh, out, ldo, I);
  return lr_launch_status();
}
