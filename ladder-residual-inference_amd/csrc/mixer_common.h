// Element access for the kernels that run in bf16 or in fp32 (template parameter: u16 = bf16 storage, float), and the
// fp32 functions they share.  Everything is computed in fp32; the storage type only decides what is read and written.
#pragma once
#include "lr_common.h"

__device__ __forceinline__ float ldf(const u16* p) { return bf_to_f(*p); }
__device__ __forceinline__ float ldf(const float* p) { return *p; }
__device__ __forceinline__ void stf(u16* p, float v) { *p = f_to_bf(v); }
__device__ __forceinline__ void stf(float* p, float v) { *p = v; }

// four consecutive elements as stored (8 or 16 bytes), and their values
template <typename T> struct Quad;
template <> struct Quad<u16> {
  uint2 r;
  __device__ __forceinline__ void zero() { r = make_uint2(0, 0); }
  __device__ __forceinline__ void load(const u16* p) { r = *reinterpret_cast<const uint2*>(p); }
  __device__ __forceinline__ void get(float* f) const {
    f[0] = bf_lo(r.x); f[1] = bf_hi(r.x); f[2] = bf_lo(r.y); f[3] = bf_hi(r.y);
  }
  __device__ __forceinline__ void put(int j, const u16* p) {
    const u32 v = *p;
    u32& w = j < 2 ? r.x : r.y;
    w = (j & 1) ? (w & 0xffffu) | (v << 16) : (w & 0xffff0000u) | v;
  }
};
template <> struct Quad<float> {
  float4 r;
  __device__ __forceinline__ void zero() { r = make_float4(0, 0, 0, 0); }
  __device__ __forceinline__ void load(const float* p) { r = *reinterpret_cast<const float4*>(p); }
  __device__ __forceinline__ void get(float* f) const { f[0] = r.x; f[1] = r.y; f[2] = r.z; f[3] = r.w; }
  __device__ __forceinline__ void put(int j, const float* p) { reinterpret_cast<float*>(&r)[j] = *p; }
};

__device__ __forceinline__ void st4(u16* p, const float* f) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf2(f[0], f[1]), pack_bf2(f[2], f[3]));
}
__device__ __forceinline__ void st4(float* p, const float* f) {
  *reinterpret_cast<float4*>(p) = make_float4(f[0], f[1], f[2], f[3]);
}

__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }

// log of sigmoid(z)^(1/tau): -softplus(-z) / tau
__device__ __forceinline__ float log_sigmoid_f(float z) { return fminf(z, 0.0f) - log1pf(expf(-fabsf(z))); }

// A single step's log-decay is cut off here: e^-60 of a state is nothing in fp32, and e^60 is still a finite factor.
constexpr float LOG_DECAY_FLOOR = -60.0f;

// Sum over the 16 lanes of a row (lanes 16 r .. 16 r + 15), every lane getting the result.
__device__ __forceinline__ float row16_sum(float v) {
  v += lr_dpp<0x128>(v);  // row_ror:8
  v += lr_dpp<0x124>(v);  // row_ror:4
  v += lr_dpp<0x4e>(v);   // quad_perm [2,3,0,1]
  v += lr_dpp<0xb1>(v);   // quad_perm [1,0,3,2]
  return v;
}
