// Grouped-query attention through a sliding window over a cache of rows [k of every kv head | v of every kv head]:
// cache [Bmax, Smax, ldc], head g's key at column g dk, its value at G dk + g dv.  Another layer may read the same cache.
//
// lr_bias_rope_cache finishes a projection [q | k | v]: bias, rotation of q and k ("rotate half" pairs), q in place, k and v
// into the cache.  Prompts and portions then attend with lr_window_attention (cache rows as they lie); single tokens with
// lr_window_decode: the window cut into ranges that run side by side, scores on the matrix cores, softmax and sums in fp32,
// the ranges merged by a second launch.
#include "mixer_common.h"

namespace {

struct RopeCache {
  void* proj;
  int64_t ld;
  const void* bias;         // [(H + 2 G) heads' columns], may be NULL
  const float* rope;        // [len, rot / 2, 2]
  const int32_t* pos;
  void* cache;              // NULL: the projection is q alone
  int rows, S, H, G, dk, dv, rot, rope_len, ldc, Smax;
  int32_t* err;
};

// A workgroup per token (few tokens: several); an item is a rotation pair, or two columns that pass.
template <typename T>
__global__ __launch_bounds__(256) void k_bias_rope_cache(const RopeCache a) {
  const int row = blockIdx.x, b = row / a.S, s = row - b * a.S;
  const int p = a.pos[s];
  if (p < 0 || p >= a.Smax || (a.rot && p >= a.rope_len)) {
    if (a.err && threadIdx.x == 0) *a.err = LR_DEV_POS_RANGE;
    return;
  }
  T* x = reinterpret_cast<T*>(a.proj) + (int64_t)row * a.ld;
  const T* bias = reinterpret_cast<const T*>(a.bias);
  const int half = a.rot >> 1, dk2 = (a.dk + 1) >> 1;
  const int heads = a.H + (a.cache ? a.G : 0);
  T* crow = a.cache ? reinterpret_cast<T*>(a.cache) + ((int64_t)b * a.Smax + p) * a.ldc : nullptr;
  auto value = [&](int c) { return ldf(x + c) + (bias ? ldf(bias + c) : 0.0f); };
  const int first = blockIdx.y * 256 + threadIdx.x, step = gridDim.y * 256;
  for (int i = first; i < heads * dk2; i += step) {
    const int h = i / dk2, j = i - h * dk2;
    T* out = h < a.H ? x + h * a.dk : crow + (h - a.H) * a.dk;
    if (j < half) {
      const float u = value(h * a.dk + j), v = value(h * a.dk + j + half);
      const float2 cs = *reinterpret_cast<const float2*>(a.rope + ((int64_t)p * half + j) * 2);
      stf(out + j, u * cs.x - v * cs.y);
      stf(out + j + half, v * cs.x + u * cs.y);
    } else {
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int c = a.rot + 2 * (j - half) + e;
        if (c < a.dk) stf(out + c, value(h * a.dk + c));
      }
    }
  }
  if (crow) {
    const int v0 = (a.H + a.G) * a.dk;
    for (int i = first; i < a.G * a.dv; i += step) stf(crow + a.G * a.dk + i, value(v0 + i));
  }
}

struct WinDecode {
  const u16* q;
  int64_t ldq;
  const u16* cache;
  const int32_t* pos;
  float *o, *ml;            // [B, H, nsplit, dv], [B, H, nsplit, 2]
  int H, G, dk, dv, ldc, Smax, window, nsplit, hblocks;
  float c2;                 // scale in base-2 exponents
};

constexpr int DKEYS = 128;  // keys per range, at most: all requested at once

// One range of one kv head, up to 16 of its query heads.  HD: a bound on both head sizes.
template <int HD>
__global__ __launch_bounds__(256) void k_window_decode(const WinDecode a) {
  constexpr int KS = HD / 32, LPK = HD / 8, KPW = 64 / LPK, NI = 32 / KPW;   // NI: value loads per wave (32 keys)
  constexpr int SCL = DKEYS + 4;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* sc = sm;                       // [16][SCL]
  float* s_m = sc + 16 * SCL;           // [16]
  float* s_l = s_m + 16;                // [16]
  float* ored = s_l + 16;               // [4][heads][HD]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g4 = lane >> 4, l16 = lane & 15;
  const int sp = blockIdx.x, kvh = blockIdx.y / a.hblocks, hb = (blockIdx.y - kvh * a.hblocks) * 16, b = blockIdx.z;
  const int share = a.H / a.G, nh = min(16, share - hb), h0 = kvh * share + hb;
  const int p = min(a.pos[0], a.Smax - 1);
  const int lo = max(0, p - a.window + 1), n = p - lo + 1;
  const int per = min(DKEYS, ((n + a.nsplit - 1) / a.nsplit + 15) & ~15);
  const int k0 = lo + sp * per, nk = min(per, p + 1 - k0);
  float* mlp = a.ml + (((int64_t)b * a.H + h0) * a.nsplit + sp) * 2;
  if (nk <= 0) {
    if (tid < nh) {
      mlp[(int64_t)tid * a.nsplit * 2] = -INFINITY;
      mlp[(int64_t)tid * a.nsplit * 2 + 1] = 0.0f;
    }
    return;
  }
  const rsrc_t rc = buffer_of(a.cache + ((int64_t)b * a.Smax + k0) * a.ldc, nk * a.ldc * 2);
  const rsrc_t rq = buffer_of(a.q + (int64_t)b * a.ldq + (int64_t)h0 * a.dk, nh * a.dk * 2);
  // wave w: keys 32 w .. 32 w + 31 of the range
  u32x4_t qf[KS], kf[2][KS], vf[NI];
#pragma unroll
  for (int k = 0; k < KS; ++k) {
    const int c = 32 * k + 8 * g4;
    qf[k] = __builtin_amdgcn_raw_buffer_load_b128(rq, l16 < nh && c < a.dk ? (l16 * a.dk + c) * 2 : NOWHERE, 0, 0);
  }
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int key = 32 * wave + 16 * t + l16, c = 32 * k + 8 * g4;
      kf[t][k] = __builtin_amdgcn_raw_buffer_load_b128(rc, key < nk && c < a.dk ? (key * a.ldc + kvh * a.dk + c) * 2 : NOWHERE, 0, 0);
    }
  const int kl = lane / LPK, dl = (lane % LPK) * 8;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int key = 32 * wave + i * KPW + kl;
    vf[i] = __builtin_amdgcn_raw_buffer_load_b128(rc, key < nk && dl < a.dv ? (key * a.ldc + a.G * a.dk + kvh * a.dv + dl) * 2 : NOWHERE, 0, 0);
  }
#pragma unroll
  for (int t = 0; t < 2; ++t) {
    f32x4_t acc = {0, 0, 0, 0};
#pragma unroll
    for (int k = 0; k < KS; ++k)
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, kf[t][k]), __builtin_bit_cast(bf16x8_t, qf[k]), acc, 0, 0, 0);
    // register i: key 32 wave + 16 t + 4 g4 + i, head l16
    const int key = 32 * wave + 16 * t + 4 * g4;
    float f[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) f[i] = key + i < nk ? acc[i] * a.c2 : -INFINITY;
    *reinterpret_cast<float4*>(&sc[l16 * SCL + key]) = make_float4(f[0], f[1], f[2], f[3]);
  }
  __syncthreads();
  for (int g = wave; g < nh; g += 4) {
    const float x0 = sc[g * SCL + lane], x1 = sc[g * SCL + 64 + lane];
    const float m = wave_max(fmaxf(x0, x1));
    const float w0 = exp2_f(x0 - m), w1 = exp2_f(x1 - m);
    sc[g * SCL + lane] = w0;
    sc[g * SCL + 64 + lane] = w1;
    const float l = wave_sum(w0 + w1);
    if (lane == 0) { s_m[g] = m; s_l[g] = l; }
  }
  __syncthreads();
  // sums: a lane owns eight columns of every KPW-th key of its wave; then over the wave's key groups and the waves
  for (int g = 0; g < nh; ++g) {
    float acc[8] = {0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      float v[8];
      unpack8(__builtin_bit_cast(uint4, vf[i]), v);
      const float w = sc[g * SCL + 32 * wave + i * KPW + kl];
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[e] = fmaf(w, v[e], acc[e]);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e)
#pragma unroll
      for (int o = LPK; o < 64; o <<= 1) acc[e] += __shfl_xor(acc[e], o, LR_WAVE);
    if (kl == 0) {
      float* d = ored + ((int64_t)wave * nh + g) * HD + dl;
      *reinterpret_cast<float4*>(d) = make_float4(acc[0], acc[1], acc[2], acc[3]);
      *reinterpret_cast<float4*>(d + 4) = make_float4(acc[4], acc[5], acc[6], acc[7]);
    }
  }
  __syncthreads();
  float* op = a.o + (((int64_t)b * a.H + h0) * a.nsplit + sp) * a.dv;
  for (int i = tid; i < nh * a.dv; i += 256) {
    const int g = i / a.dv, d = i - g * a.dv;
    float t = 0.0f;
#pragma unroll
    for (int w = 0; w < 4; ++w) t += ored[(w * nh + g) * HD + d];
    op[(int64_t)g * a.nsplit * a.dv + d] = t;
  }
  if (tid < nh) {
    mlp[(int64_t)tid * a.nsplit * 2] = s_m[tid];
    mlp[(int64_t)tid * a.nsplit * 2 + 1] = s_l[tid];
  }
}

__global__ __launch_bounds__(256) void k_window_merge(const float* __restrict__ o, const float* __restrict__ ml, u16* __restrict__ y,
                                                      int64_t ldy, int H, int dv, int nsplit) {
  const int h = blockIdx.x, b = blockIdx.y, d = threadIdx.x;
  const float* m = ml + ((int64_t)b * H + h) * nsplit * 2;
  const float* op = o + ((int64_t)b * H + h) * nsplit * dv + (d < dv ? d : 0);
  float M = -INFINITY;
#pragma unroll 8
  for (int s = 0; s < nsplit; ++s) M = fmaxf(M, m[2 * s]);
  float L = 0.0f, t = 0.0f;
#pragma unroll 8
  for (int s = 0; s < nsplit; ++s) {
    const float w = exp2_f(m[2 * s] - M), x = op[(int64_t)s * dv];   // an empty range: weight 0, nothing written there
    L = fmaf(w, m[2 * s + 1], L);
    t = fmaf(w, w > 0.0f ? x : 0.0f, t);
  }
  if (d < dv) y[(int64_t)b * ldy + h * dv + d] = f_to_bf(L > 0.0f ? t / L : 0.0f);
}

int splits(int B, int G, int hblocks, int window, int Smax) {
  const int keys = window < Smax ? window : Smax;
  const int least = (keys + DKEYS - 1) / DKEYS, most = (keys + 31) / 32;
  int n = (512 + B * G * hblocks - 1) / (B * G * hblocks);
  if (n > most) n = most;
  return n < least ? least : n;
}

template <int HD>
int launch_decode(const WinDecode& a, int B, hipStream_t s) {
  const int nh = a.H / a.G < 16 ? a.H / a.G : 16;
  const size_t lds = sizeof(float) * (16 * (DKEYS + 4) + 32 + 4 * nh * HD);
  static std::atomic<unsigned long long> raised{0};
  if (!lr_raise_lds_limit(reinterpret_cast<const void*>(&k_window_decode<HD>), lds, raised)) return LR_E_LAUNCH;
  k_window_decode<HD><<<dim3(a.nsplit, a.G * a.hblocks, B), dim3(256), lds, s>>>(a);
  return lr_launch_status();
}

}  // namespace

extern "C" int lr_bias_rope_cache(void* proj, int64_t ld, const void* bias, const float* rope, const int32_t* pos, void* cache, int B,
                                  int S, int H, int G, int dk, int dv, int rot, int rope_len, int ldc, int Smax, int dtype, int32_t* err,
                                  lr_stream_t stream) {
  LR_REQUIRE_PTR(proj);
  LR_OPTIONAL_PTR(bias);
  LR_OPTIONAL_PTR(rope);
  LR_OPTIONAL_PTR(cache);
  if (pos == nullptr || (rot > 0 && rope == nullptr)) return LR_E_NULL;
  if (B <= 0 || S <= 0 || H <= 0 || G <= 0 || H % G || dk <= 0 || dv <= 0 || rot < 0 || rot % 2 || rot > dk || Smax <= 0) return LR_E_SHAPE;
  const int64_t cols = (int64_t)H * dk + (cache ? (int64_t)G * (dk + dv) : 0);
  if (ld < cols || (cache && ldc < G * (dk + dv)) || (int64_t)B * S > 0x7fffffff) return LR_E_SHAPE;
  const RopeCache a = {proj, ld, bias, rope, pos, cache, B * S, S, H, G, dk, dv, rot, rope_len, ldc, Smax, err};
  const int items = ((H + (cache ? G : 0)) * ((dk + 1) / 2) + 255) / 256;
  const dim3 grid(a.rows, a.rows <= 64 ? (items < 16 ? items : 16) : 1);
  if (dtype == LR_BF16) k_bias_rope_cache<u16><<<grid, dim3(256), 0, (hipStream_t)stream>>>(a);
  else if (dtype == LR_F32) k_bias_rope_cache<float><<<grid, dim3(256), 0, (hipStream_t)stream>>>(a);
  else return LR_E_UNSUPPORTED;
  return lr_launch_status();
}

extern "C" size_t lr_window_decode_scratch_bytes(int B, int H, int G, int dv, int window, int Smax) {
  if (B <= 0 || H <= 0 || G <= 0 || H % G || dv <= 0 || window <= 0 || Smax <= 0) return 0;
  return sizeof(float) * (size_t)B * H * splits(B, G, (H / G + 15) / 16, window, Smax) * (dv + 2);
}

extern "C" int lr_window_decode(const void* q, int64_t ldq, const void* cache, const int32_t* pos, void* y, int64_t ldy, int B, int H,
                                int G, int dk, int dv, int ldc, int Smax, int window, float scale, void* scratch, size_t scratch_bytes,
                                lr_stream_t stream) {
  LR_REQUIRE_PTR(q);
  LR_REQUIRE_PTR(cache);
  LR_REQUIRE_PTR(y);
  LR_REQUIRE_PTR(scratch);
  if (pos == nullptr) return LR_E_NULL;
  if (B <= 0 || H <= 0 || G <= 0 || H % G || dk <= 0 || dv <= 0 || window <= 0 || Smax <= 0 || ldq < (int64_t)H * dk ||
      ldy < (int64_t)H * dv || ldc < G * (dk + dv))
    return LR_E_SHAPE;
  if (dk % 8 || dv % 8 || ldq % 8 || ldc % 8) return LR_E_ALIGN;
  const int hd = dk > dv ? dk : dv, hblocks = (H / G + 15) / 16;
  if (hd > 256 || B > 65535 || (int64_t)G * hblocks > 65535 || (int64_t)DKEYS * ldc * 2 >= 0x7fffffff) return LR_E_UNSUPPORTED;
  if (scratch_bytes < lr_window_decode_scratch_bytes(B, H, G, dv, window, Smax)) return LR_E_SHAPE;
  const int ns = splits(B, G, hblocks, window, Smax);
  float* o = reinterpret_cast<float*>(scratch);
  const WinDecode a = {(const u16*)q, ldq, (const u16*)cache, pos, o, o + (size_t)B * H * ns * dv, H, G, dk, dv, ldc, Smax, window, ns,
                       hblocks, scale * LOG2E};
  hipStream_t s = (hipStream_t)stream;
  const int rc = hd <= 64 ? launch_decode<64>(a, B, s) : hd <= 128 ? launch_decode<128>(a, B, s) : launch_decode<256>(a, B, s);
  if (rc != LR_OK) return rc;
  k_window_merge<<<dim3(H, B), dim3((dv + 63) / 64 * 64), 0, s>>>(o, a.ml, (u16*)y, ldy, H, dv, ns);
  return lr_launch_status();
}
