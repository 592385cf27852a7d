// lm_device.h - device helpers of the layer-list models' kernels (lm_latent.hip, lm_mixers.hip): block sums, bf16 packing, operand stores
#pragma once
#include "lm_latent.h"

__device__ __forceinline__ float lat_block_sum(float v, float* red) {          // any block of whole waves; every thread gets the total
    v = wave_sum_dpp(v);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    const int nw = blockDim.x >> 6;
    float t = 0.0f;
    for (int i = 0; i < nw; ++i) t += red[i];
    __syncthreads();
    return t;
}
__device__ __forceinline__ void load4_bf16(const bf16_t* p, float (&o)[4]) {
    const uint2 q = *reinterpret_cast<const uint2*>(p);
    o[0] = bf16_to_f32((bf16_t)(q.x & 0xffffu)); o[1] = bf16_to_f32((bf16_t)(q.x >> 16));
    o[2] = bf16_to_f32((bf16_t)(q.y & 0xffffu)); o[3] = bf16_to_f32((bf16_t)(q.y >> 16));
}
__device__ __forceinline__ uint2 pack4_bf16(const float (&v)[4]) {
    return make_uint2((uint32_t)f32_to_bf16(v[0]) | ((uint32_t)f32_to_bf16(v[1]) << 16), (uint32_t)f32_to_bf16(v[2]) | ((uint32_t)f32_to_bf16(v[3]) << 16));
}
// four consecutive columns k .. k + 3 (k % 4 == 0) of operand row m
__device__ __forceinline__ void operand_store4(const Operand& h, int m, int k, const float (&v)[4]) {
    if (h.kind == OPK_F32) *reinterpret_cast<float4*>((float*)h.p + (size_t)m * h.ld + k) = make_float4(v[0], v[1], v[2], v[3]);
    else {
        bf16_t* o = (bf16_t*)h.p + (h.kind == OPK_PACKED ? xpk_index(m, k, h.MT) : (size_t)m * h.ld + k);
        *reinterpret_cast<uint2*>(o) = pack4_bf16(v);
    }
}
__device__ __forceinline__ void operand_store1(const Operand& h, int m, int k, float v) {
    if (h.kind == OPK_F32) ((float*)h.p)[(size_t)m * h.ld + k] = v;
    else ((bf16_t*)h.p)[h.kind == OPK_PACKED ? xpk_index(m, k, h.MT) : (size_t)m * h.ld + k] = f32_to_bf16(v);
}

__device__ __forceinline__ void put(float* p, float v) { *p = v; }
__device__ __forceinline__ void put(bf16_t* p, float v) { *p = f32_to_bf16(v); }
__device__ __forceinline__ float get(const float* p) { return *p; }
__device__ __forceinline__ float get(const bf16_t* p) { return bf16_to_f32(*p); }

__device__ __forceinline__ void put4(float* p, const float (&v)[4]) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
__device__ __forceinline__ void put4(bf16_t* p, const float (&v)[4]) { *reinterpret_cast<uint2*>(p) = pack4_bf16(v); }
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }
__device__ __forceinline__ bf16x8_t lds_frag(const bf16_t* p) { return *reinterpret_cast<const bf16x8_t*>(p); }
