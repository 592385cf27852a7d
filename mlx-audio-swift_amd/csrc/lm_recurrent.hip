// lm_recurrent.hip - the recurrences of lm_mixers.h on the matrix cores (bf16): gated linear recurrence (decode step, prompt chunks) and attention with
// a decayed outer-product state (decode step on the vector units, prompt chunks on the matrix cores).  States, decays, gates and sums are float32;
// float32 values that enter a product do so as bf16 hi + lo pairs.
#include "lm_mixers.h"
#include "lm_device.h"
#include "lm_recurrent.h"
#include <math.h>

__device__ __forceinline__ uint32_t rec_pair(float a, float b) { return (uint32_t)f32_to_bf16(a) | ((uint32_t)f32_to_bf16(b) << 16); }

// ============================================================================ gated linear recurrence: gates
// Block = 64 output channels of one block of channels (a wave: one 16-row tile of both gate matrices) x 64 consecutive tokens of one request (decode
// steps: recur_step_block).  The convolution's outputs u of 128 channels at a time come into LDS as hi and lo fragments; the
// channels the block's own outputs belong to come last and stay for the epilogue, which scans the 64 tokens - 16 on the lanes of a DPP row, the tiles one
// after the other - and leaves, per token, the state reached from zero (loc) and the product of the decays (dec) since the chunk's start.
#define REC_KC 128
template <int S>
__device__ __forceinline__ float rec_shr(float v, float before) {              // lane i of a row of 16: v of lane i - S; the first S lanes: before
    return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(__builtin_bit_cast(int, before), __builtin_bit_cast(int, v), 0x110 | S, 0xF, 0xF, false));
}
template <int S>
__device__ __forceinline__ void rec_scan_step(float& a, float& b) {
    const float pa = rec_shr<S>(a, 1.0f), pb = rec_shr<S>(b, 0.0f);
    b += a * pb;
    a *= pa;
}
// VEC: a block's channels are a multiple of 4.  TAPS4: at most four taps - a thread's four tokens follow each other and share the inputs they reach back to
template <bool VEC, bool TAPS4>
__global__ void __launch_bounds__(256, 2) k_recur_gates(RecurDims D, RecurParams p, const RecurChunk* __restrict__ chunks, float* __restrict__ loc, float* __restrict__ dec,
                                                        float* __restrict__ carry0) {
    constexpr int MT = RECUR_CHUNK / 16;
    __shared__ __attribute__((aligned(16))) bf16_t us[REC_KC / 32][2][MT][512];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = lane & 15, lq = lane >> 4;
    const int slices = (D.nt + 3) >> 2, b = blockIdx.y / slices, sl = blockIdx.y - b * slices;
    const int tile = sl * 4 + wave, KT = D.np >> 5;
    const int ch0 = b * D.n;                                                   // first channel of the block
    const RecurChunk c = chunks[blockIdx.x];
    const int m0 = c.rows.row0, nrows = c.rows.n;
    const int grp = tid & 15, r0 = tid >> 4;                                   // staging: 8 channels, rows 4 r0 .. + 3
    f32x4_t ar[MT], ag[MT];
#pragma unroll
    for (int t = 0; t < MT; ++t) ar[t] = ag[t] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
    const int nc = (D.np + REC_KC - 1) / REC_KC, own = (sl * 64) / REC_KC;
    const bf16x8_t* wr = reinterpret_cast<const bf16x8_t*>(p.ra) + ((size_t)(b * D.nt + min(tile, D.nt - 1)) * KT) * 64 + lane;
    const bf16x8_t* wg = reinterpret_cast<const bf16x8_t*>(p.ri) + ((size_t)(b * D.nt + min(tile, D.nt - 1)) * KT) * 64 + lane;
    for (int cc = 0; cc < nc; ++cc) {
        const int kc = cc == nc - 1 ? own : (cc < own ? cc : cc + 1);          // every chunk of channels once, the block's own last
        bf16x8_t fr[REC_KC / 32], fg[REC_KC / 32];
#pragma unroll
        for (int k = 0; k < REC_KC / 32; ++k) {
            const int kt = min(kc * (REC_KC / 32) + k, KT - 1);
            fr[k] = wr[(size_t)kt * 64]; fg[k] = wg[(size_t)kt * 64];
        }
        if (cc) __syncthreads();
        const int i0 = kc * REC_KC + grp * 8;                                  // channel inside the block
        // clamped places, no branches: channels past the block and rows past the end are dropped behind the sum
        auto load8 = [&](const float* v) {
            f32x8_t x;
            if constexpr (VEC) {
                const int a0 = min(i0, D.n - 4), a1 = min(i0 + 4, D.n - 4);
                x = __builtin_shufflevector(*reinterpret_cast<const f32x4_t*>(v + ch0 + a0), *reinterpret_cast<const f32x4_t*>(v + ch0 + a1), 0, 1, 2, 3, 4, 5, 6, 7);
            } else {
#pragma unroll
                for (int j = 0; j < 8; ++j) x[j] = v[ch0 + min(i0 + j, D.n - 1)];
            }
            return x;
        };
        const f32x8_t xb = load8(p.bias_x), u0 = load8(p.conv_b32);
        auto input = [&](int r) {                                              // of the convolution at row r of the chunk (below 0: before it)
            const int at = min(r, nrows - 1), q = c.rows.pos0 + at;
            const bool here = q >= c.span_pos0;                                // this pass's rows, or what earlier ones left
            f32x8_t x = load8(here ? p.proj + (size_t)(m0 + at) * p.ld + p.ox : p.hist + ((size_t)c.rows.seq * D.taps + max(q, 0) % D.taps) * D.W);
            if (here) x += xb;
#pragma unroll
            for (int j = 0; j < 8; ++j) x[j] = q < 0 ? 0.0f : x[j];
            return x;
        };
        f32x8_t u[MT];
#pragma unroll
        for (int t = 0; t < MT; ++t) u[t] = u0;
        if constexpr (TAPS4) {
            f32x8_t w[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                w[i] = load8(p.conv_t + (size_t)max(D.taps - 1 - i, 0) * D.W);
                if (i >= D.taps) w[i] = (f32x8_t){0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            }
#pragma unroll
            for (int k = 0; k < MT + 3; ++k) {                                 // row r0 MT + k - 3 is what tap t - (k - 3) of token t reads
                const f32x8_t x = input(r0 * MT + k - 3);
#pragma unroll
                for (int t = 0; t < MT; ++t)
                    if (t - (k - 3) >= 0 && t - (k - 3) < 4) u[t] += w[t - (k - 3)] * x;
            }
        } else {
            for (int i = 0; i < D.taps; ++i) {
                const f32x8_t w = load8(p.conv_t + (size_t)(D.taps - 1 - i) * D.W);
#pragma unroll
                for (int t = 0; t < MT; ++t) u[t] += w * input(r0 * MT + t - i);
            }
        }
#pragma unroll
        for (int t = 0; t < MT; ++t) {
            const int r = r0 * MT + t;
            bf16x8_t hi, lo;
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const float v = r < nrows && i0 + j < D.n ? u[t][j] : 0.0f;
                const bf16_t h = f32_to_bf16(v);
                hi[j] = (short)h;
                lo[j] = (short)f32_to_bf16(v - bf16_to_f32(h));
            }
            const int kt = grp >> 2, at = ((grp & 3) * 16 + (r & 15)) * 8;
            *reinterpret_cast<bf16x8_t*>(&us[kt][0][r >> 4][at]) = hi;
            *reinterpret_cast<bf16x8_t*>(&us[kt][1][r >> 4][at]) = lo;
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < REC_KC / 32; ++k) {
            if (kc * (REC_KC / 32) + k >= KT) continue;
#pragma unroll
            for (int t = 0; t < MT; ++t) {
                const bf16x8_t hi = lds_frag(&us[k][0][t][lane * 8]), lo = lds_frag(&us[k][1][t][lane * 8]);
                ar[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fr[k], hi, ar[t], 0, 0, 0);
                ar[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fr[k], lo, ar[t], 0, 0, 0);
                ag[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fg[k], hi, ag[t], 0, 0, 0);
                ag[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fg[k], lo, ag[t], 0, 0, 0);
            }
        }
    }
    if (tile >= D.nt) return;
    // ---- epilogue: lane = channels i .. i + 3 of rows t * 16 + li
    const int i = tile * 16 + lq * 4, ch = ch0 + i, nv = min(4, D.n - i);
    if (nv <= 0) return;
    float cf[4], rb[4], gb[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const int q = ch + min(e, nv - 1);
        cf[e] = p.c[q]; rb[e] = bf16_to_f32(p.ra_b[q]); gb[e] = bf16_to_f32(p.ri_b[q]);
    }
    float ca[4] = {1.f, 1.f, 1.f, 1.f}, cb[4] = {0.f, 0.f, 0.f, 0.f};          // product and state up to the tile (prompt)
#pragma unroll
    for (int t = 0; t < MT; ++t) {
        const int r = t * 16 + li, m = m0 + r;
        const int at = (((i & 31) >> 3) * 16 + li) * 8 + (i & 7), kt = (i & (REC_KC - 1)) >> 5;
        const uint2 h = *reinterpret_cast<const uint2*>(&us[kt][0][t][at]), l = *reinterpret_cast<const uint2*>(&us[kt][1][t][at]);
        const uint32_t hw[2] = {h.x, h.y}, lw[2] = {l.x, l.y};
        float a[4], x[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int sh = 16 * (e & 1);
            const float u = bf16_to_f32((bf16_t)((hw[e >> 1] >> sh) & 0xffffu)) + bf16_to_f32((bf16_t)((lw[e >> 1] >> sh) & 0xffffu));
            const float la = -cf[e] * rec_sigmoid(ar[t][e] + rb[e]);
            a[e] = rec_exp(la);
            x[e] = rec_complement(a[e], la) * rec_sigmoid(ag[t][e] + gb[e]) * u;
        }
        const bool on = r < nrows;
        float A[4], B[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            float pa = on ? a[e] : 1.0f, pb = on ? x[e] : 0.0f;
            rec_scan_step<1>(pa, pb);
            rec_scan_step<2>(pa, pb);
            rec_scan_step<4>(pa, pb);
            rec_scan_step<8>(pa, pb);
            B[e] = pb + pa * cb[e];
            A[e] = pa * ca[e];
            ca[e] = __shfl(A[e], lane | 15, 64);
            cb[e] = __shfl(B[e], lane | 15, 64);
        }
        if (!on) continue;
        float *lp = loc + (size_t)m * D.W + ch, *dp = dec + (size_t)m * D.W + ch;
        if (VEC) {
            *reinterpret_cast<float4*>(lp) = make_float4(B[0], B[1], B[2], B[3]);
            *reinterpret_cast<float4*>(dp) = make_float4(A[0], A[1], A[2], A[3]);
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e) if (e < nv) { lp[e] = B[e]; dp[e] = A[e]; }
        }
    }
    if (c.index == 0 && li == 0)                                               // what the span starts from (its last chunk overwrites the state)
        for (int e = 0; e < nv; ++e) carry0[(size_t)c.span * D.W + ch + e] = c.span_pos0 == 0 ? 0.0f : p.state[(size_t)c.rows.seq * D.W + ch + e];
}
template <bool VEC>
__global__ void __launch_bounds__(256) k_recur_step(RecurDims D, RecurParams p, int rows) {
    __shared__ RecurStepLds<1> L;
    recur_step_block<VEC, 1>(D, p, rows, blockIdx.x, L);
}
void launch_recur_step(const RecurDims& D, const RecurParams& p, int rows, hipStream_t s) {
    MIS_REQUIRE(p.rows.pos && !p.rows.seq, MIS_ERR_GENERATION_FAILED, "gated recurrence step: bad layout");
    if (D.n % 4 == 0) hipLaunchKernelGGL((k_recur_step<true>), dim3(recur_step_blocks(D, rows, 1)), dim3(256), 0, s, D, p, rows);
    else hipLaunchKernelGGL((k_recur_step<false>), dim3(recur_step_blocks(D, rows, 1)), dim3(256), 0, s, D, p, rows);
}
// chunk: state = loc + dec * (state before the chunk), times the other branch; the chunks before it in the span give that state
__global__ void __launch_bounds__(256) k_recur_apply(RecurDims D, RecurParams p, const RecurChunk* __restrict__ chunks, const float* __restrict__ loc,
                                                     const float* __restrict__ dec, const float* __restrict__ carry0) {
    const RecurChunk c = chunks[blockIdx.x];
    const int ch = blockIdx.y * 64 + (threadIdx.x & 63), part = threadIdx.x >> 6;
    if (ch >= D.W) return;
    float h = carry0[(size_t)c.span * D.W + ch];
    const int first = c.rows.row0 - c.index * RECUR_CHUNK;
#pragma unroll 8
    for (int k = 0; k < c.index; ++k) {
        const size_t e = ((size_t)first + k * RECUR_CHUNK + RECUR_CHUNK - 1) * D.W + ch;
        h = dec[e] * h + loc[e];
    }
    const float yb = bf16_to_f32(p.bias[p.oy + ch]);
    const int t1 = min((part + 1) * (RECUR_CHUNK / 4), c.rows.n);
    float S = h;
#pragma unroll 4
    for (int t = part * (RECUR_CHUNK / 4); t < t1; ++t) {
        const size_t m = c.rows.row0 + t;
        S = dec[m * D.W + ch] * h + loc[m * D.W + ch];
        operand_store1(p.out, (int)m, p.col0 + ch, S * rec_gelu_tanh(p.proj[m * p.ld + p.oy + ch] + yb) * p.out_scale);
    }
    if (c.last && part == (c.rows.n - 1) / (RECUR_CHUNK / 4)) {
        p.state[(size_t)c.rows.seq * D.W + ch] = S;
        const int end = c.rows.pos0 + c.rows.n;
        for (int q = max(c.span_pos0, end - D.taps + 1); q < end; ++q)
            p.hist[((size_t)c.rows.seq * D.taps + q % D.taps) * D.W + ch] = p.proj[(size_t)(c.rows.row0 + q - c.rows.pos0) * p.ld + p.ox + ch] + p.bias_x[ch];
    }
}
void launch_recur_prefill(const RecurDims& D, const RecurParams& p, const RecurChunk* chunks, int n_chunks, float* loc, float* dec, float* carry0, hipStream_t s) {
    const dim3 grid(n_chunks, D.B * cdiv(D.nt, 4));
#define REC_GATES(V, T) hipLaunchKernelGGL((k_recur_gates<V, T>), grid, dim3(256), 0, s, D, p, chunks, loc, dec, carry0)
    if (D.n % 4 == 0) { if (D.taps <= 4) REC_GATES(true, true); else REC_GATES(true, false); }
    else { if (D.taps <= 4) REC_GATES(false, true); else REC_GATES(false, false); }
#undef REC_GATES
    hipLaunchKernelGGL(k_recur_apply, dim3(n_chunks, cdiv(D.W, 64)), dim3(256), 0, s, D, p, chunks, loc, dec, carry0);
}

__global__ void k_conv_tables(const bf16_t* __restrict__ conv, const bf16_t* __restrict__ conv_b, const bf16_t* __restrict__ bias_x, float* __restrict__ conv_t,
                              float* __restrict__ conv_b32, float* __restrict__ bias_x32, int W, int taps) {
    const int ch = blockIdx.x * blockDim.x + threadIdx.x;
    if (ch >= W) return;
    for (int i = 0; i < taps; ++i) conv_t[(size_t)i * W + ch] = bf16_to_f32(conv[(size_t)ch * taps + i]);
    conv_b32[ch] = bf16_to_f32(conv_b[ch]);
    bias_x32[ch] = bf16_to_f32(bias_x[ch]);
}
void launch_conv_tables(const bf16_t* conv, const bf16_t* conv_b, const bf16_t* bias_x, float* conv_t, float* conv_b32, float* bias_x32, int W, int taps, hipStream_t s) {
    hipLaunchKernelGGL(k_conv_tables, dim3(cdiv(W, 256)), dim3(256), 0, s, conv, conv_b, bias_x, conv_t, conv_b32, bias_x32, W, taps);
}

// ============================================================================ decayed outer-product state, decode step
// Block = 64 value columns of one head of one row; 16 threads x 4 columns, 16 shares of the key dimensions.  The state - most of the launch's bytes - is
// requested before the projections and written back from the same registers.
template <int DR>
__global__ void __launch_bounds__(256) k_decay_step(DecayDims D, DecayParams p) {
    __shared__ float sq[DR * 16], sk[DR * 16];
    __shared__ float red[16][68];
    const int hd = blockIdx.x / D.ns, sl = blockIdx.x - hd * D.ns, m = blockIdx.y, tid = threadIdx.x, c4 = (tid & 15) * 4, dg = tid >> 4;
    const bool fresh = p.spans.pos[m] == 0;
    float* state = p.state + ((size_t)m * D.H + hd) * D.D * D.Es + sl * 64 + c4;
    f32x4_t S[DR];
#pragma unroll
    for (int j = 0; j < DR; ++j) S[j] = __builtin_nontemporal_load(reinterpret_cast<const f32x4_t*>(state + (size_t)min(dg + 16 * j, D.D - 1) * D.Es));
    __builtin_amdgcn_sched_barrier(0);
    if (p.spans.on && !p.spans.on[m]) return;
    const float* row = p.proj + (size_t)m * p.ld;
    for (int i = tid; i < DR * 16; i += 256) {
        sq[i] = i < D.D ? rec_silu(row[p.oq + hd * D.D + i]) : 0.0f;
        sk[i] = i < D.D ? rec_silu(row[p.ok + hd * D.D + i]) : 0.0f;
    }
    f32x4_t v, o = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) { const int c = sl * 64 + c4 + e; v[e] = c < D.E ? rec_silu(row[p.ov + hd * D.E + c]) : 0.0f; }
    const float dc = p.decay[hd];
    __syncthreads();
#pragma unroll
    for (int j = 0; j < DR; ++j) {
        const int i = dg + 16 * j;
        if (i >= D.D) continue;
        const float k = sk[i], q = sq[i];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            S[j][e] = fresh ? k * v[e] : dc * S[j][e] + k * v[e];
            o[e] += S[j][e] * q;
        }
        __builtin_nontemporal_store(S[j], reinterpret_cast<f32x4_t*>(state + (size_t)i * D.Es));
    }
    *reinterpret_cast<f32x4_t*>(&red[dg][c4]) = o;
    __syncthreads();
    if (tid < 64) {
        float a = 0.0f;
#pragma unroll
        for (int i = 0; i < 16; ++i) a += red[i][tid];
        const int c = sl * 64 + tid;
        if (c < D.E) operand_store1(p.out, m, hd * D.E + c, a * bf16_to_f32(p.norm[hd * D.E + c]) * rec_sigmoid(row[p.og + hd * D.E + c]));
        const float ss = wave_sum(c < D.E ? a * a : 0.0f);
        if (tid == 0) p.ss[(size_t)m * D.H * D.ns + hd * D.ns + sl] = ss;
    }
}
bool decay_mfma_ok(const DecayDims& D) { return D.D <= 256; }
void launch_decay_step(const DecayDims& D, const DecayParams& p, int rows, hipStream_t s) {
    MIS_REQUIRE(decay_mfma_ok(D) && !p.spans.span && p.spans.pos, MIS_ERR_GENERATION_FAILED, "decayed state step: bad layout");
    const dim3 grid(D.H * D.ns, rows), block(256);
    if (D.D <= 64) hipLaunchKernelGGL((k_decay_step<4>), grid, block, 0, s, D, p);
    else if (D.D <= 128) hipLaunchKernelGGL((k_decay_step<8>), grid, block, 0, s, D, p);
    else hipLaunchKernelGGL((k_decay_step<16>), grid, block, 0, s, D, p);
}

// ============================================================================ decayed outer-product state, prompt
// Block = 64 value columns of one head of one request, walking its tokens in chunks of 64; wave w holds the state of columns 16 w .. + 15 in registers as
// accumulators (rows: key dimensions).  Per chunk, with t, s places in the chunk and c the decay:
//   o_t = c^(t + 1) S^T q_t + sum over s <= t of c^(t - s) (q_t . k_s) v_s;      S = c^n S + sum_s k_s (c^(n - 1 - s) v_s)^T
// A pair of state tiles is, in a lane, dimensions 4 q .. + 3 and 16 + 4 q .. + 3 of its column: the state enters S^T q straight from the accumulators (as
// hi + lo), the queries are read in that order; the pair weights go into the next product the same way (see lm_grouped.hip), keys in that order.
// q, k, v and the gate come as bf16 behind their activation (the projection's epilogue), everything that carries a decay is hi + lo.  The next chunk's
// rows are in flight meanwhile.
// A long request is cut into segments that run beside each other: a first launch (ENDS) takes every segment but the last from a zero state - the first one
// from the request's - to its end and leaves that state; the second starts segment i from the ends before it, E_0 c^(..) + .. + E_{i - 1}.  The slot of
// the last segment's end holds the state the request came with (the last segment overwrites it).
#define DCP_C 64
// VEC: the heads' sizes are multiples of 4
template <int DT, bool VEC, bool ENDS>
__global__ void __launch_bounds__(256, DT <= 4 ? 2 : 1) k_decay_prefill(DecayDims D, DecayParams p, const DecaySegment* __restrict__ segs, float* __restrict__ ends) {
    constexpr int DP = DT * 32, QS = DP + 8, TS = DCP_C + 8, NQ = (DP / 4 * 16 + 255) / 256;
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    bf16_t* sq = reinterpret_cast<bf16_t*>(lds);                               // [64][QS] queries
    bf16_t* sk = sq + DCP_C * QS;                                              // [64][QS] keys
    bf16_t* st = sk + DCP_C * QS;                                              // [DP][TS] keys, transposed
    bf16_t* sv = st + DP * TS;                                                 // [64][TS] values, transposed
    float* pw = reinterpret_cast<float*>(sv + 64 * TS) + DCP_C;                // c^i for i = 0 .. 64, zero for i = -64 .. -1 (pairs out of order)
    float* ssq = pw + 68;                                                      // [4][64]
    const int hd = blockIdx.x / D.ns, sl = blockIdx.x - hd * D.ns, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = lane & 15, lq = lane >> 4;
    const DecaySegment sg = segs[blockIdx.y];
    const RowSpan sp = sg.rows;
    const bool last = sg.index == sg.count - 1;
    if (ENDS && sg.count == 1) return;
    const float dc = p.decay[hd];
    if (tid <= 2 * DCP_C) pw[tid - DCP_C] = tid < DCP_C ? 0.0f : powf(dc, (float)(tid - DCP_C));
    float* state = p.state + ((size_t)sp.seq * D.H + hd) * D.D * D.Es + sl * 64 + wave * 16 + li;
    f32x4_t S[2 * DT];
#pragma unroll
    for (int t = 0; t < 2 * DT; ++t) S[t] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
    // (dimensions past the head meet zero queries and keys)
    const size_t slot = (size_t)D.H * D.D * D.Es;                              // a segment's end
    float* end = ends + (size_t)blockIdx.y * slot + (size_t)hd * D.D * D.Es + sl * 64 + wave * 16 + li;
    auto load_state = [&](const float* src, float scale) {                     // S = scale S + state
#pragma unroll
        for (int t = 0; t < 2 * DT; ++t)
#pragma unroll
            for (int e = 0; e < 4; ++e) S[t][e] = scale * S[t][e] + src[(size_t)min(t * 16 + lq * 4 + e, D.D - 1) * D.Es];
    };
    auto store_state = [&](float* dst) {
#pragma unroll
        for (int t = 0; t < 2 * DT; ++t)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int d = t * 16 + lq * 4 + e;
                if (d < D.D) dst[(size_t)d * D.Es] = S[t][e];
            }
    };
    if (ENDS) {
        if (sg.span_pos0 > 0 && (sg.index == 0 || last)) load_state(state, 0.0f);
        if (last) { store_state(end); return; }                                // the state the request came with
    } else if (sg.count == 1) { if (sp.pos0 > 0) load_state(state, 0.0f); }
    else if (sg.index == 0) { if (sp.pos0 > 0) load_state(end + (size_t)(sg.count - 1) * slot, 0.0f); }
    else {
        const float cs = powf(dc, (float)sg.length);
        for (int k = 0; k < sg.index; ++k) load_state(end - (size_t)(sg.index - k) * slot, cs);
    }
    float nrm[4];                                                              // norm weights of this wave's outputs
#pragma unroll
    for (int e = 0; e < 4; ++e) nrm[e] = bf16_to_f32(p.norm[hd * D.E + min(sl * 64 + wave * 16 + lq * 4 + e, D.E - 1)]);
    // an item of the staging: 4 tokens x 4 columns
    // an unconditional load of a clamped place each (behind a branch every load would be waited for alone); `only` drops what lies outside
    uint2 rq[NQ][4], rk[NQ][4], rv[4];
    auto load4 = [&](const bf16_t* q, int col, int limit) {
        if constexpr (VEC) return *reinterpret_cast<const uint2*>(q + min(col, limit - 4));
        else return make_uint2(q[min(col, limit - 1)] | (uint32_t)q[min(col + 1, limit - 1)] << 16, q[min(col + 2, limit - 1)] | (uint32_t)q[min(col + 3, limit - 1)] << 16);
    };
    auto only = [&](uint2 x, int col, int limit, bool on) {
        if (!on) return make_uint2(0, 0);
        if constexpr (VEC) return col < limit ? x : make_uint2(0, 0);
        else return make_uint2((col < limit ? x.x & 0xffffu : 0) | (col + 1 < limit ? x.x & 0xffff0000u : 0), (col + 2 < limit ? x.y & 0xffffu : 0) | (col + 3 < limit ? x.y & 0xffff0000u : 0));
    };
    auto fetch = [&](int c0) {
        const int n = sp.n - c0;
#pragma unroll
        for (int i = 0; i < NQ; ++i) {
            const int it = tid + 256 * i, t4 = it / (DP / 4) * 4, col = (it % (DP / 4)) * 4;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const bf16_t* row = p.act + (size_t)(sp.row0 + c0 + min(t4 + j, n - 1)) * p.ld;
                if (!ENDS) rq[i][j] = load4(row + p.oq + hd * D.D, col, D.D);
                rk[i][j] = load4(row + p.ok + hd * D.D, col, D.D);
            }
        }
        const int t4 = (tid >> 4) * 4, col = (tid & 15) * 4;
#pragma unroll
        for (int j = 0; j < 4; ++j) rv[j] = load4(p.act + (size_t)(sp.row0 + c0 + min(t4 + j, n - 1)) * p.ld + p.ov + hd * D.E, sl * 64 + col, D.E);
    };
    // 4 tokens x 4 columns -> column rows of 4 tokens
    auto turn = [&](const uint2 (&r)[4], bf16_t* dst) {
        auto pick = [](uint32_t a, uint32_t b, bool high) { return __builtin_amdgcn_perm(b, a, high ? 0x07060302u : 0x05040100u); };
        *reinterpret_cast<uint2*>(dst) = make_uint2(pick(r[0].x, r[1].x, false), pick(r[2].x, r[3].x, false));
        *reinterpret_cast<uint2*>(dst + TS) = make_uint2(pick(r[0].x, r[1].x, true), pick(r[2].x, r[3].x, true));
        *reinterpret_cast<uint2*>(dst + 2 * TS) = make_uint2(pick(r[0].y, r[1].y, false), pick(r[2].y, r[3].y, false));
        *reinterpret_cast<uint2*>(dst + 3 * TS) = make_uint2(pick(r[0].y, r[1].y, true), pick(r[2].y, r[3].y, true));
    };
    fetch(0);
    for (int c0 = 0; c0 < sp.n; c0 += DCP_C) {
        const int n = min(DCP_C, sp.n - c0);
        __syncthreads();                                                       // everyone is done with the chunk before
#pragma unroll
        for (int i = 0; i < NQ; ++i) {
            const int it = tid + 256 * i, t4 = it / (DP / 4) * 4, col = (it % (DP / 4)) * 4;
            if (t4 >= DCP_C) continue;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                rk[i][j] = only(rk[i][j], col, D.D, t4 + j < n);
                if (ENDS) continue;
                rq[i][j] = only(rq[i][j], col, D.D, t4 + j < n);
                *reinterpret_cast<uint2*>(sq + (t4 + j) * QS + col) = rq[i][j];
                *reinterpret_cast<uint2*>(sk + (t4 + j) * QS + col) = rk[i][j];
            }
            turn(rk[i], st + col * TS + t4);
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) rv[j] = only(rv[j], sl * 64 + (tid & 15) * 4, D.E, (tid >> 4) * 4 + j < n);
        turn(rv, sv + ((tid & 15) * 4) * TS + (tid >> 4) * 4);
        if (c0 + DCP_C < sp.n) fetch(c0 + DCP_C);
        const int vc = sl * 64 + wave * 16 + lq * 4;
        __syncthreads();
        auto two = [](const bf16_t* a, const bf16_t* b) {                      // 4 + 4 elements
            const uint2 x = *reinterpret_cast<const uint2*>(a), y = *reinterpret_cast<const uint2*>(b);
            const uint4 z = make_uint4(x.x, x.y, y.x, y.y);
            return __builtin_bit_cast(bf16x8_t, z);
        };
        const bf16_t* vr = sv + (wave * 16 + li) * TS + lq * 4;
        if constexpr (!ENDS) {
            bf16x8_t sh[DT], sl_[DT];
#pragma unroll
            for (int k = 0; k < DT; ++k)
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    const float x = S[2 * k + (j >> 2)][j & 3];
                    const bf16_t h = f32_to_bf16(x);
                    sh[k][j] = (short)h;
                    sl_[k][j] = (short)f32_to_bf16(x - bf16_to_f32(h));
                }
#pragma unroll 1
            for (int qt = 0; qt * 16 < n; ++qt) {
                const uint2 gate = load4(p.act + (size_t)(sp.row0 + c0 + min(qt * 16 + li, n - 1)) * p.ld + p.og + hd * D.E, vc, D.E);
                const bf16_t* qr = sq + (qt * 16 + li) * QS;
                f32x4_t o = (f32x4_t){0.f, 0.f, 0.f, 0.f}, ol = o;
#pragma unroll
                for (int k = 0; k < DT; ++k) {
                    const bf16x8_t q = two(qr + k * 32 + lq * 4, qr + k * 32 + 16 + lq * 4);
                    o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sh[k], q, o, 0, 0, 0);
                    ol = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sl_[k], q, ol, 0, 0, 0);
                }
                o = (o + ol) * pw[qt * 16 + li + 1];
                bf16x8_t q[DT];
#pragma unroll
                for (int k = 0; k < DT; ++k) q[k] = lds_frag(qr + k * 32 + lq * 8);
#pragma unroll 1
                for (int kp = 0; kp <= qt / 2; ++kp) {
                    f32x4_t a0 = (f32x4_t){0.f, 0.f, 0.f, 0.f}, a1 = a0;
                    const bf16_t *k0 = sk + (kp * 32 + li) * QS + lq * 8, *k1 = k0 + 16 * QS;
#pragma unroll
                    for (int k = 0; k < DT; ++k) {
                        a0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lds_frag(k0 + k * 32), q[k], a0, 0, 0, 0);
                        a1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lds_frag(k1 + k * 32), q[k], a1, 0, 0, 0);
                    }
                    bf16x8_t ph, pl;
#pragma unroll
                    for (int j = 0; j < 8; ++j) {
                        const int d = qt * 16 + li - (kp * 32 + (j >> 2) * 16 + lq * 4 + (j & 3));
                        const float x = (j < 4 ? a0[j & 3] : a1[j & 3]) * pw[d];
                        const bf16_t h = f32_to_bf16(x);
                        ph[j] = (short)h;
                        pl[j] = (short)f32_to_bf16(x - bf16_to_f32(h));
                    }
                    const bf16x8_t v = two(vr + kp * 32, vr + kp * 32 + 16);
                    o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, ph, o, 0, 0, 0);
                    o = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pl, o, 0, 0, 0);
                }
                // rows of o: value columns, columns: tokens
                const int t = qt * 16 + li;
                float ss = (o[0] * o[0] + o[1] * o[1]) + (o[2] * o[2] + o[3] * o[3]);
                ss += __shfl_xor(ss, 16, 64);
                ss += __shfl_xor(ss, 32, 64);
                if (lq == 0) ssq[wave * 64 + t] = ss;
                if (t < n) {
                    const float g[4] = {bf16_to_f32((bf16_t)(gate.x & 0xffffu)), bf16_to_f32((bf16_t)(gate.x >> 16)), bf16_to_f32((bf16_t)(gate.y & 0xffffu)),
                                        bf16_to_f32((bf16_t)(gate.y >> 16))};
                    const size_t m = sp.row0 + c0 + t;
                    float x[4];
#pragma unroll
                    for (int e = 0; e < 4; ++e) x[e] = vc + e < D.E ? o[e] * nrm[e] * g[e] : 0.0f;
                    bf16_t* dst = (bf16_t*)p.out.p + m * p.out.ld + hd * D.E + vc;
                    if constexpr (VEC) { if (vc < D.E) *reinterpret_cast<uint2*>(dst) = pack4_bf16(x); }
                    else {
#pragma unroll
                        for (int e = 0; e < 4; ++e) if (vc + e < D.E) dst[e] = f32_to_bf16(x[e]);
                    }
                }
            }
        }
        // state
        const float pn = pw[n];
#pragma unroll
        for (int t = 0; t < 2 * DT; ++t) S[t] *= pn;
#pragma unroll
        for (int kp = 0; kp < 2; ++kp) {
            const bf16x8_t v = two(vr + kp * 32, vr + kp * 32 + 16);
            bf16x8_t vh, vl;
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const float x = bf16_to_f32((bf16_t)v[j]) * pw[max(n - 1 - (kp * 32 + (j >> 2) * 16 + lq * 4 + (j & 3)), 0)];
                const bf16_t h = f32_to_bf16(x);
                vh[j] = (short)h;
                vl[j] = (short)f32_to_bf16(x - bf16_to_f32(h));
            }
#pragma unroll
            for (int t = 0; t < 2 * DT; ++t) {
                const bf16_t* kr = st + (t * 16 + li) * TS + kp * 32 + lq * 4;
                const bf16x8_t k = two(kr, kr + 16);
                S[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, vh, S[t], 0, 0, 0);
                S[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, vl, S[t], 0, 0, 0);
            }
        }
        if (ENDS) continue;
        __syncthreads();
        if (tid < n) p.ss[(size_t)(sp.row0 + c0 + tid) * D.H * D.ns + hd * D.ns + sl] = (ssq[tid] + ssq[64 + tid]) + (ssq[128 + tid] + ssq[192 + tid]);
    }
    if (ENDS) store_state(end);
    else if (last) store_state(state);
}
int decay_segment_rows(const DecayDims& D, int rows, int spans) {
    const int per = cdiv(rows, spans), blocks = D.H * D.ns * spans;            // segments of at least eight chunks, until the launch fills the chip
    const int segs = std::max(1, std::min(per / (8 * DCP_C), cdiv(384, blocks)));
    return (int)round_up(cdiv(per, segs), DCP_C);
}
void launch_decay_prefill(const DecayDims& D, const DecayParams& p, const DecaySegment* segs, int n_segs, bool cut, float* ends, hipStream_t s) {
    MIS_REQUIRE(decay_mfma_ok(D) && p.act && segs && (!cut || ends) && p.out.kind == OPK_ROWS && p.out.ld % 4 == 0, MIS_ERR_GENERATION_FAILED, "decayed state prompt: bad layout");
    const dim3 grid(D.H * D.ns, n_segs), block(256);
    const bool vec = D.D % 4 == 0 && D.E % 4 == 0;
#define DCP(T) do { if (vec) DCPV(T, true); else DCPV(T, false); } while (0)
#define DCPV(T, V) do { if (cut) DCPE(T, V, true); DCPE(T, V, false); } while (0)
#define DCPE(T, V, X) do {                                                                                                                               \
        const size_t lds = (size_t)(2 * DCP_C * (T * 32 + 8) + T * 32 * (DCP_C + 8) + 64 * (DCP_C + 8)) * 2 + (DCP_C + 68 + 256) * 4;                       \
        static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&k_decay_prefill<T, V, X>), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024); \
        HIP_CHECK(attr);                                                                                                                                   \
        hipLaunchKernelGGL((k_decay_prefill<T, V, X>), grid, block, lds, s, D, p, segs, ends); } while (0)
    const int t = cdiv(D.D, 32);
    if (t == 1) DCP(1); else if (t == 2) DCP(2); else if (t <= 4) DCP(4); else DCP(8);
#undef DCP
#undef DCPV
#undef DCPE
}
