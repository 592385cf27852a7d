// lm_recurrent.h - device parts of the gated recurrence that more than one kernel file uses (lm_recurrent.hip, lm_grouped.hip)
#pragma once
#include "lm_mixers.h"
#include "lm_device.h"

// float32 on the hardware's base-2 exponential, reciprocal and square root (each within an ulp or two)
#define REC_LOG2E 1.4426950408889634f
__device__ __forceinline__ float rec_exp(float z) { return __builtin_amdgcn_exp2f(z * REC_LOG2E); }
__device__ __forceinline__ float rec_sigmoid(float z) { return __builtin_amdgcn_rcpf(1.0f + rec_exp(-z)); }
__device__ __forceinline__ float rec_silu(float z) { return z * rec_sigmoid(z); }
// 0.5 (1 + tanh y) = sigmoid(2 y)
__device__ __forceinline__ float rec_gelu_tanh(float z) { return z * rec_sigmoid(1.5957691216057308f * (z + 0.044715f * z * z * z)); }
// sqrt(1 - a^2) for a = e^la, la <= 0: near la = 0 by the series of 1 - e^t, which the difference would cancel away
__device__ __forceinline__ float rec_complement(float a, float la) {
    const float t = 2.0f * la;
    const float series = -t * (1.0f + t * (0.5f + t * (0.16666667f + t * (0.041666667f + t * (0.0083333333f + t * 0.0013888889f)))));
    return __builtin_amdgcn_sqrtf(t > -0.25f ? series : 1.0f - a * a);
}
typedef float f32x8_t __attribute__((ext_vector_type(8)));

// ---- decode step of the gated recurrence: block = 16 output channels of a block of channels, 16 rows; its four waves share the products' columns.  A wave
// computes the convolution outputs its columns need straight into hi and lo fragments (lane: 8 channels of a row); the waves' sums meet in LDS, then a
// thread finishes one (row, channel): gates, state, the other branch.
// (PARTS: such tiles per block, four waves each.)
template <int PARTS>
struct RecurStepLds { float red[PARTS][4][2][64][4]; };
static inline int recur_step_blocks(const RecurDims& D, int rows, int parts) { return cdiv((int64_t)D.B * D.nt * ((rows + 15) / 16), parts); }
// VEC: a block's channels are a multiple of 4
template <bool VEC, int PARTS>
__device__ __forceinline__ void recur_step_block(const RecurDims& D, const RecurParams& p, int rows, int block, RecurStepLds<PARTS>& lds) {
    const int tid = threadIdx.x & 255, part = threadIdx.x >> 8, lane = tid & 63, wave = tid >> 6, li = lane & 15, lq = lane >> 4;
    const int tiles = D.B * D.nt * ((rows + 15) / 16), want = block * PARTS + part, bi = min(want, tiles - 1);
    auto& red = lds.red[part];
    const int mt = bi / (D.B * D.nt), t = bi - mt * D.B * D.nt, b = t / D.nt, tile = t - b * D.nt, ch0 = b * D.n, KT = D.np >> 5;
    // ---- what the finishing thread needs, requested first
    const int fm = mt * 16 + (tid >> 4), fi = tile * 16 + (tid & 15), fmc = min(fm, rows - 1), ch = ch0 + min(fi, D.n - 1);
    const int pos_f = p.rows.pos[fmc];
    const bool on = want < tiles && fm < rows && fi < D.n && (!p.rows.on || p.rows.on[fmc]);
    const float* prow = p.proj + (size_t)fmc * p.ld;
    float* sp = p.state + (size_t)fmc * D.W + ch;
    const float s_old = *sp, x_now = prow[p.ox + ch] + p.bias_x[ch], y_raw = prow[p.oy + ch] + bf16_to_f32(p.bias[p.oy + ch]);
    const float cf = p.c[ch], rb = bf16_to_f32(p.ra_b[ch]), gb = bf16_to_f32(p.ri_b[ch]);
    float u_own = p.conv_b32[ch] + p.conv_t[(size_t)(D.taps - 1) * D.W + ch] * x_now;
    for (int i = 1; i < D.taps; ++i) {
        const int q = pos_f - i;
        const float x = p.hist[((size_t)fmc * D.taps + max(q, 0) % D.taps) * D.W + ch];
        u_own += q < 0 ? 0.0f : p.conv_t[(size_t)(D.taps - 1 - i) * D.W + ch] * x;
    }
    // ---- products
    const int m = min(mt * 16 + li, rows - 1), pos = p.rows.pos[m];
    f32x4_t ar = (f32x4_t){0.f, 0.f, 0.f, 0.f}, ag = ar, br = ar, bg = ar;
    const bf16x8_t* wr = reinterpret_cast<const bf16x8_t*>(p.ra) + (size_t)t * KT * 64 + lane;
    const bf16x8_t* wg = reinterpret_cast<const bf16x8_t*>(p.ri) + (size_t)t * KT * 64 + lane;
    for (int k = wave; k < KT; k += 4) {
        const bf16x8_t fr = wr[(size_t)k * 64], fg = wg[(size_t)k * 64];
        const int i0 = k * 32 + lq * 8;
        auto load8 = [&](const float* q) {                                     // (clamped places: channels past the block are dropped below)
            f32x8_t x;
            if constexpr (VEC) {
                const int a0 = min(i0, D.n - 4), a1 = min(i0 + 4, D.n - 4);
                x = __builtin_shufflevector(*reinterpret_cast<const f32x4_t*>(q + ch0 + a0), *reinterpret_cast<const f32x4_t*>(q + ch0 + a1), 0, 1, 2, 3, 4, 5, 6, 7);
            } else {
#pragma unroll
                for (int j = 0; j < 8; ++j) x[j] = q[ch0 + min(i0 + j, D.n - 1)];
            }
            return x;
        };
        f32x8_t u = load8(p.conv_b32) + load8(p.conv_t + (size_t)(D.taps - 1) * D.W) * (load8(p.proj + (size_t)m * p.ld + p.ox) + load8(p.bias_x));
#pragma unroll 3
        for (int i = 1; i < D.taps; ++i) {
            const int q = pos - i;
            const f32x8_t w = load8(p.conv_t + (size_t)(D.taps - 1 - i) * D.W), x = load8(p.hist + ((size_t)m * D.taps + max(q, 0) % D.taps) * D.W);
#pragma unroll
            for (int j = 0; j < 8; ++j) u[j] += q < 0 ? 0.0f : w[j] * x[j];
        }
        bf16x8_t hi, lo;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const float v = i0 + j < D.n ? u[j] : 0.0f;
            const bf16_t h = f32_to_bf16(v);
            hi[j] = (short)h;
            lo[j] = (short)f32_to_bf16(v - bf16_to_f32(h));
        }
        ar = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fr, hi, ar, 0, 0, 0);
        br = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fr, lo, br, 0, 0, 0);
        ag = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fg, hi, ag, 0, 0, 0);
        bg = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fg, lo, bg, 0, 0, 0);
    }
    *reinterpret_cast<f32x4_t*>(red[wave][0][lane]) = ar + br;
    *reinterpret_cast<f32x4_t*>(red[wave][1][lane]) = ag + bg;
    __syncthreads();
    if (!on) return;
    // ---- one (row, channel) per thread: accumulator row = channel, column = row
    const int at = ((tid & 15) >> 2) * 16 + (tid >> 4), e = tid & 3;
    const float zr = (red[0][0][at][e] + red[1][0][at][e]) + (red[2][0][at][e] + red[3][0][at][e]);
    const float zg = (red[0][1][at][e] + red[1][1][at][e]) + (red[2][1][at][e] + red[3][1][at][e]);
    const float la = -cf * rec_sigmoid(zr + rb), a = rec_exp(la);
    const float in = rec_complement(a, la) * rec_sigmoid(zg + gb) * u_own;
    const float S = pos_f == 0 ? in : a * s_old + in;
    *sp = S;
    p.hist[((size_t)fm * D.taps + pos_f % D.taps) * D.W + ch] = x_now;         // (a slot no row reads in this step)
    operand_store1(p.out, fm, p.col0 + ch, S * rec_gelu_tanh(y_raw) * p.out_scale);
}
