// lm_grouped.hip - grouped attention of lm_mixers.h on the matrix cores (bf16): prompt tiles and decode shares over the fragment caches.
//
// Both kernels compute S^T = K q^T on 16 x 16 tiles (rows: keys, columns: queries - positions of one head in a prompt, heads of one group in a decode
// step) and O^T = V^T P^T.  A pair of score tiles leaves a lane the weights of keys 4 q .. + 3 and 16 + 4 q .. + 3 of its column, and the value
// fragments hold the keys in that order: the weights go from the accumulators into the next product without leaving the lane.  Scores and softmax are
// float32, base 2; the weights enter as bf16 hi + lo.  The sink is a key-less term of the running sum: the sum starts with it.
#include "lm_mixers.h"
#include "lm_device.h"
#include "lm_recurrent.h"
#include <math.h>

#define GRP_LOG2E 1.4426950408889634f
__device__ __forceinline__ float grp_exp2(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ bool grp_sees(const GroupedDims& D, int pos, int key) {
    return (key <= pos) & ((D.window <= 0) | (pos - key < D.window) | (key < D.keep));
}
// steps of 32 keys that a query (a range of queries) may see: [0, kept) and [s0, s1]
struct GrpSteps { int kept, s0, s1; __device__ int count() const { return kept + s1 - s0 + 1; } __device__ int at(int i) const { return i < kept ? i : s0 + i - kept; } };
__device__ __forceinline__ GrpSteps grp_steps(const GroupedDims& D, int pos_lo, int pos_hi) {
    GrpSteps r;
    r.s0 = D.window > 0 ? max(0, pos_lo - D.window + 1) >> 5 : 0;
    r.s1 = pos_hi >> 5;
    r.kept = min((D.keep + 31) >> 5, r.s0);
    return r;
}
// weights of a pair of score tiles -> bf16 hi and lo fragments
__device__ __forceinline__ void grp_split(const float (&w)[8], bf16x8_t& hi, bf16x8_t& lo) {
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        const bf16_t h = f32_to_bf16(w[j]);
        hi[j] = (short)h;
        lo[j] = (short)f32_to_bf16(w[j] - bf16_to_f32(h));
    }
}

// ============================================================================ prompt pass
// Block = up to 64 queries of one request and up to four heads of one group; a wave = 32 queries of one head.  The 32 keys of a step - KT pairs of key
// fragments and VT value fragments, contiguous in the caches - come into LDS by DMA, two buffers, one barrier per step.
// EXACT: the heads have KT and VT tiles, not fewer (no guards in the loop)
template <int KT, int VT, bool EXACT>
__global__ void __launch_bounds__(512, 2) k_grouped_attn_prefill(GroupedDims D, GroupedAttn p, const RowSpan* __restrict__ tiles, int ipb) {
    __shared__ __attribute__((aligned(1024))) bf16_t buf[2][(2 * KT + VT) * 512];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = blockDim.x >> 6, li = lane & 15, lq = lane >> 4;
    const RowSpan t = tiles[gridDim.x - 1 - blockIdx.x];                       // (a request's last queries see the most keys: they start first)
    const int g = blockIdx.y, R = D.H / D.G, kt_n = EXACT ? KT : D.Dp >> 5, vt_n = EXACT ? VT : D.Ep >> 4;
    const int item = blockIdx.z * ipb + wave, hd = g * R + min(item >> 1, R - 1), q0 = (item & 1) * 32;
    const bool live = item < 2 * R && q0 < t.n;                                // (a wave without queries only helps to stage)
    const int nq = min(32, t.n - q0), p_lo = t.pos0 + q0, p_hi = p_lo + nq - 1;
    const GrpSteps st = grp_steps(D, t.pos0, t.pos0 + t.n - 1);
    const bf16_t* kc = (const bf16_t*)p.kc + ((size_t)t.seq * D.G + g) * p.Smax * D.Dp;
    const bf16_t* vc = (const bf16_t*)p.vc + ((size_t)t.seq * D.G + g) * p.Smax * D.Ep;
    auto stage = [&](int b, int s) {
        const bf16_t *ks = kc + (size_t)s * 32 * D.Dp, *vs = vc + (size_t)s * 32 * D.Ep;
        for (int f = wave; f < 2 * kt_n + vt_n; f += nw) {
            const bf16_t* src = f < 2 * kt_n ? ks + (size_t)f * 512 : vs + (size_t)(f - 2 * kt_n) * 512;
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(src + lane * 8),
                                             (__attribute__((address_space(3))) void*)&buf[b][(f < 2 * kt_n ? f : 2 * KT + f - 2 * kt_n) * 512], 16, 0, 0);
        }
    };
    stage(0, st.at(0));
    bf16x8_t q[2][KT];
    int pos[2];
#pragma unroll
    for (int c = 0; c < 2; ++c) {
        const int r = live ? min(c * 16 + li, nq - 1) : 0;
        pos[c] = p_lo + c * 16 + li;
        const bf16_t* qr = (const bf16_t*)p.q + ((size_t)(live ? t.row0 + q0 + r : t.row0) * D.H + hd) * D.Dp + lq * 8;
#pragma unroll
        for (int k = 0; k < KT; ++k) q[c][k] = *reinterpret_cast<const bf16x8_t*>(qr + min(k, kt_n - 1) * 32);
    }
    f32x4_t o[2][VT];
#pragma unroll
    for (int c = 0; c < 2; ++c)
#pragma unroll
        for (int v = 0; v < VT; ++v) o[c][v] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
    const float sc = D.scale * GRP_LOG2E, sink = bf16_to_f32(p.sink[hd]) * GRP_LOG2E;
    float mx[2] = {sink, sink}, ls[2] = {lq == 0 ? 1.0f : 0.0f, lq == 0 ? 1.0f : 0.0f};      // ls: this lane's keys only
    const int n = st.count();
    for (int i = 0; i < n; ++i) {
        __syncthreads();                                                       // step i has landed; the other buffer is free
        if (i + 1 < n) stage((i + 1) & 1, st.at(i + 1));
        const int k0 = st.at(i) * 32;
        if (!live || k0 > p_hi) continue;                                      // (wave-uniform)
        if (D.window > 0 && p_lo - (k0 + 31) >= D.window && k0 >= D.keep) continue;
        const bf16_t* b = buf[i & 1];
        f32x4_t s[2][2];
#pragma unroll
        for (int c = 0; c < 2; ++c) s[c][0] = s[c][1] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < KT; ++k) {
            if (k >= kt_n) continue;
            const bf16x8_t a0 = lds_frag(b + (size_t)k * 512 + lane * 8), a1 = lds_frag(b + (size_t)(kt_n + k) * 512 + lane * 8);
#pragma unroll
            for (int c = 0; c < 2; ++c) {
                s[c][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a0, q[c][k], s[c][0], 0, 0, 0);
                s[c][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a1, q[c][k], s[c][1], 0, 0, 0);
            }
        }
        const bool all = k0 + 31 <= p_lo && (D.window <= 0 || p_hi - k0 < D.window || k0 + 31 < D.keep);
        bf16x8_t ph[2], pl[2];
#pragma unroll
        for (int c = 0; c < 2; ++c) {
            float w[8], tm = -INFINITY;
#pragma unroll
            for (int h = 0; h < 2; ++h)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    w[h * 4 + e] = s[c][h][e] * sc;
                    if (!all && !grp_sees(D, pos[c], k0 + h * 16 + lq * 4 + e)) w[h * 4 + e] = -INFINITY;
                    tm = fmaxf(tm, w[h * 4 + e]);
                }
            tm = fmaxf(tm, __shfl_xor(tm, 16, 64));
            tm = fmaxf(tm, __shfl_xor(tm, 32, 64));
            if (__any(tm > mx[c])) {
                const float mn = fmaxf(mx[c], tm), alpha = grp_exp2(mx[c] - mn);
                mx[c] = mn;
                ls[c] *= alpha;
#pragma unroll
                for (int v = 0; v < VT; ++v) o[c][v] *= alpha;
            }
            float add = 0.0f;
#pragma unroll
            for (int j = 0; j < 8; ++j) { w[j] = grp_exp2(w[j] - mx[c]); add += w[j]; }
            ls[c] += add;
            grp_split(w, ph[c], pl[c]);
        }
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            if (v >= vt_n) continue;
            const bf16x8_t a = lds_frag(b + (size_t)(2 * KT + v) * 512 + lane * 8);
#pragma unroll
            for (int c = 0; c < 2; ++c) {
                o[c][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, ph[c], o[c][v], 0, 0, 0);
                o[c][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, pl[c], o[c][v], 0, 0, 0);
            }
        }
    }
    if (!live) return;
#pragma unroll
    for (int c = 0; c < 2; ++c) {
        float l = ls[c];
        l += __shfl_xor(l, 16, 64);
        l += __shfl_xor(l, 32, 64);
        const float r = p.out_scale / l;
        if (c * 16 + li >= nq) continue;
        const int m = t.row0 + q0 + c * 16 + li;
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            const int col = v * 16 + lq * 4;
            const float x[4] = {o[c][v][0] * r, o[c][v][1] * r, o[c][v][2] * r, o[c][v][3] * r};
            if ((D.E & 3) == 0) { if (col < D.E) operand_store4(p.out, m, hd * D.E + col, x); }
            else {
#pragma unroll
                for (int e = 0; e < 4; ++e) if (col + e < D.E) operand_store1(p.out, m, hd * D.E + col + e, x[e]);
            }
        }
    }
}
// Projections of a pass -> query rows and caches.  Queries and keys: LPV lanes a vector, four dimensions a lane.  Values (the blocks behind n_qk): four
// positions x four columns a thread, whole groups of four positions as one store each.
__global__ void __launch_bounds__(256) k_grouped_rows_prefill(GroupedDims D, GroupedRows p, const RowSpan* __restrict__ tiles, int rows, int n_qk, int LPV, int vblocks) {
    const int tid = threadIdx.x;
    if ((int)blockIdx.x < n_qk) {
        const int vec = (blockIdx.x * 256 + tid) / LPV, l = tid & (LPV - 1), HG = D.H + D.G, m = min(vec / HG, rows - 1), a = vec % HG;
        const bool is_q = a < D.H, on = vec < rows * HG, in = 4 * l < D.D;
        const int o = is_q ? p.oq + a * D.D : p.ok + (a - D.H) * D.D, i = 4 * l, ic = in ? i : 0, half = D.rot >> 1;
        const int pos = p.rows.pos[m], seq = p.rows.seq ? p.rows.seq[m] : m;
        const float4 x4 = *reinterpret_cast<const float4*>(p.proj + (size_t)m * p.ld + o + ic);
        float b[4], w[4], x[4] = {x4.x, x4.y, x4.z, x4.w};
        load4_bf16(p.bias + o + ic, b);
        load4_bf16((is_q ? p.qn : p.kn) + ic, w);
        const bool lowp = i < half, turn = i < D.rot;
        const int ri = turn ? (lowp ? i : i - half) : 0;
        float4 c = make_float4(1.f, 1.f, 1.f, 1.f), s = make_float4(0.f, 0.f, 0.f, 0.f);
        if (half) { c = *reinterpret_cast<const float4*>(p.rope_cos + (size_t)pos * half + ri); s = *reinterpret_cast<const float4*>(p.rope_sin + (size_t)pos * half + ri); }
        float ss = 0.0f;
#pragma unroll
        for (int e = 0; e < 4; ++e) { x[e] = in ? x[e] + b[e] : 0.0f; ss += x[e] * x[e]; }
        for (int d = LPV >> 1; d > 0; d >>= 1) ss += __shfl_xor(ss, d, 64);
        const float inv = 1.0f / sqrtf(ss / (float)D.D + D.eps);
        const float cv[4] = {c.x, c.y, c.z, c.w}, sv[4] = {s.x, s.y, s.z, s.w};
        const int other = (tid & 63) + (turn ? (lowp ? half >> 2 : -(half >> 2)) : 0);
        float v[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            x[e] *= inv * w[e];
            const float y = __shfl(x[e], other, 64);
            v[e] = turn ? (lowp ? x[e] * cv[e] - y * sv[e] : x[e] * cv[e] + y * sv[e]) : x[e];
        }
        if (!on || i >= D.Dp) return;
        bf16_t* dst = is_q ? (bf16_t*)p.q + ((size_t)m * D.H + a) * D.Dp + i
                           : (bf16_t*)p.kc + ((((size_t)seq * D.G + a - D.H) * (p.Smax >> 4) + (pos >> 4)) * (D.Dp >> 5) + (i >> 5)) * 512 + (((i & 31) >> 3) * 16 + (pos & 15)) * 8 + (i & 7);
        *reinterpret_cast<uint2*>(dst) = pack4_bf16(v);
        return;
    }
    const int vb = blockIdx.x - n_qk, tile = vb / vblocks, e4 = D.E >> 2, it = (vb - tile * vblocks) * 256 + tid;
    const RowSpan t = tiles[tile];
    const int col = (it % e4) * 4, g = (it / e4) % D.G, p4 = (t.pos0 & ~3) + 4 * (it / (e4 * D.G));
    if (p4 >= t.pos0 + t.n) return;
    float x[4][4], b[4];
    load4_bf16(p.bias + p.ov + g * D.E + col, b);
#pragma unroll
    for (int k = 0; k < 4; ++k) {
        const int q = min(max(p4 + k, t.pos0), t.pos0 + t.n - 1);
        const float4 f = *reinterpret_cast<const float4*>(p.proj + (size_t)(t.row0 + q - t.pos0) * p.ld + p.ov + g * D.E + col);
        x[k][0] = f.x + b[0]; x[k][1] = f.y + b[1]; x[k][2] = f.z + b[2]; x[k][3] = f.w + b[3];
    }
    const bool whole = p4 >= t.pos0 && p4 + 3 < t.pos0 + t.n;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const int i = col + e;
        bf16_t* dst = (bf16_t*)p.vc + ((((size_t)t.seq * D.G + g) * (p.Smax >> 5) + (p4 >> 5)) * (D.Ep >> 4) + (i >> 4)) * 512 + (((p4 & 15) >> 2) * 16 + (i & 15)) * 8 +
                      ((p4 >> 4) & 1) * 4;
        const float v[4] = {x[0][e], x[1][e], x[2][e], x[3][e]};
        if (whole) *reinterpret_cast<uint2*>(dst) = pack4_bf16(v);
        else
#pragma unroll
            for (int k = 0; k < 4; ++k)
                if (p4 + k >= t.pos0 && p4 + k < t.pos0 + t.n) dst[k] = f32_to_bf16(v[k]);
    }
}
void launch_grouped_rows_prefill(const GroupedDims& D, const GroupedRows& p, const RowSpan* tiles, int n_tiles, int rows, hipStream_t s) {
    if (D.D % 4 || D.E % 4 || D.rot % 8 || D.Dp > 256 || p.f32 || p.rows.on) { launch_grouped_rows(D, p, rows, s); return; }
    MIS_REQUIRE(p.rows.pos && p.Smax % 32 == 0 && D.rot <= D.D && D.H % D.G == 0 && p.ld % 4 == 0, MIS_ERR_GENERATION_FAILED, "grouped attention: bad layout");
    int lpv = 8;
    while (lpv * 4 < D.Dp) lpv *= 2;
    const int n_qk = cdiv((int64_t)rows * (D.H + D.G) * lpv, 256), vblocks = cdiv((int64_t)(GROUPED_QT / 4 + 1) * D.G * (D.E / 4), 256);
    hipLaunchKernelGGL(k_grouped_rows_prefill, dim3(n_qk + n_tiles * vblocks), dim3(256), 0, s, D, p, tiles, rows, n_qk, lpv, vblocks);
}

bool grouped_mfma_ok(const GroupedDims& D) { return D.Dp <= 256 && D.Ep <= 256; }
void launch_grouped_attn_prefill(const GroupedDims& D, const GroupedAttn& p, const RowSpan* tiles, int n_tiles, hipStream_t s) {
    MIS_REQUIRE(grouped_mfma_ok(D) && !p.f32 && p.Smax % 32 == 0 && p.out.kind == OPK_ROWS && p.out.ld % 4 == 0, MIS_ERR_GENERATION_FAILED, "grouped attention: bad layout");
    const int items = 2 * (D.H / D.G);
    int ipb = std::min(items, 8);                                              // waves per block: they share the staged keys
    while (items > 8 && ipb > 4 && items % ipb) --ipb;
    const dim3 grid(n_tiles, D.G, cdiv(items, ipb)), block(64 * ipb);
    const int kt = D.Dp / 32, vt = D.Ep / 16;
#define GRP_PF(K, V, X) hipLaunchKernelGGL((k_grouped_attn_prefill<K, V, X>), grid, block, 0, s, D, p, tiles, ipb)
    if (kt == 2 && vt == 4) GRP_PF(2, 4, true);
    else if (kt == 4 && vt == 8) GRP_PF(4, 8, true);
    else if (kt <= 2 && vt <= 4) GRP_PF(2, 4, false);
    else if (kt <= 4 && vt <= 8) GRP_PF(4, 8, false);
    else GRP_PF(8, 16, false);
#undef GRP_PF
}

// ============================================================================ decode step
// Block = one row, up to 16 heads of one group, one share of the row's steps; its eight waves take the share's steps in turn, each with its own running
// softmax, and meet in LDS once.  The block norms and rotates its heads' queries itself; the current token's key and value never come from the cache: its
// score and value join when the waves meet (last share), the sink with the first share.  The last share's block of a group's first head tile also
// appends the token to the caches - for the NEXT step.
#define GRP_NW 8
template <int VT>
struct GrpDecodeLds { float q[16][260]; float k[260], v[260]; float m[GRP_NW][16], l[GRP_NW][16], self[16]; float acc[GRP_NW][16][VT * 16 + 4]; };
template <int KT, int VT, bool EXACT>
__device__ __forceinline__ void grouped_decode_block(const GroupedDims& D, const GroupedRows& r, const GroupedAttn& p, const GroupedShares& sh, int rows, int bx, int g, int bz,
                                                     GrpDecodeLds<VT>& L) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, li = lane & 15, lq = lane >> 4;
    const int m = bx % rows, sp = bx / rows, R = D.H / D.G, kt_n = EXACT ? KT : D.Dp >> 5, vt_n = EXACT ? VT : D.Ep >> 4;
    const int a0 = bz * 16, na = min(16, R - a0), h0 = g * R + a0;             // heads h0 .. h0 + na - 1
    const int pos = r.rows.pos[m], half = D.rot >> 1;
    if (r.rows.on && !r.rows.on[m]) return;                                    // block-uniform
    const GrpSteps st = grp_steps(D, pos, pos);
    const int n = st.count(), per = (n + sh.S - 1) / sh.S, i0 = min(sp * per, n), i1 = min(i0 + per, n);
    const bool first = sp == 0, last = sp == sh.S - 1;
    const bf16_t* kc = (const bf16_t*)p.kc + ((size_t)m * D.G + g) * p.Smax * D.Dp;
    const bf16_t* vc = (const bf16_t*)p.vc + ((size_t)m * D.G + g) * p.Smax * D.Ep;
    bf16x8_t ka[2][KT], va[VT];
    auto fetch_k = [&](int s) {
        const bf16_t* ks = kc + (size_t)s * 32 * D.Dp + lane * 8;
#pragma unroll
        for (int k = 0; k < KT; ++k) {
            ka[0][k] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8_t*>(ks + (size_t)min(k, kt_n - 1) * 512));
            ka[1][k] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8_t*>(ks + (size_t)(kt_n + min(k, kt_n - 1)) * 512));
        }
    };
    auto fetch_v = [&](int s) {
        const bf16_t* vs = vc + (size_t)s * 32 * D.Ep + lane * 8;
#pragma unroll
        for (int v = 0; v < VT; ++v) va[v] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8_t*>(vs + (size_t)min(v, vt_n - 1) * 512));
    };
    // ---- queries (and, last share, the token's key and value): bias, norm, rotation; a wave per vector.  Its projections are requested before the wave's
    // first keys (loads return in order)
    const float *cs = r.rope_cos + (size_t)pos * half, *sn = r.rope_sin + (size_t)pos * half;
    const float* row = r.proj + (size_t)m * r.ld;
    const int n_vec = na + (last ? 2 : 0);                                     // heads, key, value
    float x[4], xb[4], xw[4];                                                  // sizes <= 256: four dimensions a lane
    auto load_vec = [&](int a) {
        const int o = a < na ? r.oq + (h0 + a) * D.D : (a == na ? r.ok + g * D.D : r.ov + g * D.E), size = a <= na ? D.D : D.E;
        const bf16_t* w = a < na ? r.qn : r.kn;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int i = min(lane + 64 * j, size - 1);
            x[j] = row[o + i]; xb[j] = bf16_to_f32(r.bias[o + i]); xw[j] = bf16_to_f32(w[min(i, D.D - 1)]);
        }
    };
    if (wave < n_vec) load_vec(wave);
    float rc[2], rs[2];                                                        // half <= 128: two pairs a lane
#pragma unroll
    for (int j = 0; j < 2; ++j) { const int i = min(lane + 64 * j, max(half - 1, 0)); rc[j] = cs[i]; rs[j] = sn[i]; }
    __builtin_amdgcn_sched_barrier(0);
    if (i0 + wave < i1) { fetch_k(st.at(i0 + wave)); fetch_v(st.at(i0 + wave)); }
    __builtin_amdgcn_sched_barrier(0);
    for (int a = wave; a < n_vec; a += GRP_NW) {
        if (a != wave) load_vec(a);
        const int size = a <= na ? D.D : D.E;
        float ss = 0.0f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            x[j] = lane + 64 * j < size ? x[j] + xb[j] : 0.0f;
            ss += x[j] * x[j];
        }
        if (a == na + 1) {                                                     // value
#pragma unroll
            for (int j = 0; j < 4; ++j) if (lane + 64 * j < D.Ep) L.v[lane + 64 * j] = bf16_round_f32(x[j]);
            continue;
        }
        const float inv = 1.0f / sqrtf(wave_sum_dpp(ss) / (float)D.D + D.eps);
        float* dst = a < na ? L.q[a] : L.k;
#pragma unroll
        for (int j = 0; j < 4; ++j) if (lane + 64 * j < D.Dp) dst[lane + 64 * j] = x[j] * inv * xw[j];
        __builtin_amdgcn_wave_barrier();                                       // (one wave's LDS accesses stay in order)
#pragma unroll
        for (int j = 0; j < 2; ++j) {                                          // rotation in place
            const int i = lane + 64 * j;
            if (i >= half) continue;
            const float u = dst[i], v = dst[i + half];
            dst[i] = u * rc[j] - v * rs[j];
            dst[i + half] = v * rc[j] + u * rs[j];
        }
    }
    for (int i = threadIdx.x + na * 260; i < 16 * 260; i += 64 * GRP_NW) L.q[0][i] = 0.0f;           // columns past the heads
    __syncthreads();
    if (last) {
        if (a0 == 0) {
            bf16_t *kd = (bf16_t*)r.kc + ((size_t)m * D.G + g) * p.Smax * D.Dp, *vd = (bf16_t*)r.vc + ((size_t)m * D.G + g) * p.Smax * D.Ep;
            for (int i = threadIdx.x; i < D.Dp; i += 64 * GRP_NW)
                kd[((size_t)(pos >> 4) * kt_n + (i >> 5)) * 512 + (((i & 31) >> 3) * 16 + (pos & 15)) * 8 + (i & 7)] = f32_to_bf16(L.k[i]);
            for (int i = threadIdx.x; i < D.Ep; i += 64 * GRP_NW)
                vd[((size_t)(pos >> 5) * vt_n + (i >> 4)) * 512 + (((pos & 15) >> 2) * 16 + (i & 15)) * 8 + ((pos >> 4) & 1) * 4 + (pos & 3)] = f32_to_bf16(L.v[i]);
        }
        for (int a = wave; a < na; a += GRP_NW) {                              // score of the token with itself, on the values the cache will hold
            float d = 0.0f;
            for (int i = lane; i < D.D; i += 64) d += bf16_round_f32(L.q[a][i]) * bf16_round_f32(L.k[i]);
            d = wave_sum_dpp(d);
            if (lane == 0) L.self[a] = d * D.scale * GRP_LOG2E;
        }
    }
    bf16x8_t q[KT];
#pragma unroll
    for (int k = 0; k < KT; ++k) {
        const float* x = &L.q[li][min(k, kt_n - 1) * 32 + lq * 8];
#pragma unroll
        for (int e = 0; e < 8; ++e) q[k][e] = (short)f32_to_bf16(x[e]);
    }
    f32x4_t o[VT];
#pragma unroll
    for (int v = 0; v < VT; ++v) o[v] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
    const float sc = D.scale * GRP_LOG2E;
    float mx = -1e30f, ls = 0.0f;
    for (int i = i0 + wave; i < i1; i += GRP_NW) {
        const int k0 = st.at(i) * 32;
        f32x4_t s0 = (f32x4_t){0.f, 0.f, 0.f, 0.f}, s1 = s0;
#pragma unroll
        for (int k = 0; k < KT; ++k) {
            if (k >= kt_n) continue;
            s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka[0][k], q[k], s0, 0, 0, 0);
            s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka[1][k], q[k], s1, 0, 0, 0);
        }
        if (i + GRP_NW < i1) fetch_k(st.at(i + GRP_NW));
        __builtin_amdgcn_sched_barrier(0);
        float w[8], tm = -1e30f;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const int key = k0 + (j >> 2) * 16 + lq * 4 + (j & 3);
            const bool on = key != pos && grp_sees(D, pos, key);
            w[j] = on ? (j < 4 ? s0[j & 3] : s1[j & 3]) * sc : -INFINITY;
            tm = fmaxf(tm, w[j]);
        }
        tm = fmaxf(tm, __shfl_xor(tm, 16, 64));
        tm = fmaxf(tm, __shfl_xor(tm, 32, 64));
        if (__any(tm > mx)) {
            const float mn = fmaxf(mx, tm), alpha = grp_exp2(mx - mn);
            mx = mn;
            ls *= alpha;
#pragma unroll
            for (int v = 0; v < VT; ++v) o[v] *= alpha;
        }
        float add = 0.0f;
#pragma unroll
        for (int j = 0; j < 8; ++j) { w[j] = grp_exp2(w[j] - mx); add += w[j]; }
        ls += add;
        bf16x8_t ph, pl;
        grp_split(w, ph, pl);
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            if (v >= vt_n) continue;
            o[v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va[v], ph, o[v], 0, 0, 0);
            o[v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va[v], pl, o[v], 0, 0, 0);
        }
        if (i + GRP_NW < i1) fetch_v(st.at(i + GRP_NW));
        __builtin_amdgcn_sched_barrier(0);
    }
    // ---- the waves meet: common maximum (with the sink and the token itself), sums, values; a thread per head and four columns
    ls += __shfl_xor(ls, 16, 64);
    ls += __shfl_xor(ls, 32, 64);
    if (lq == 0) { L.m[wave][li] = mx; L.l[wave][li] = ls; }
#pragma unroll
    for (int v = 0; v < VT; ++v) *reinterpret_cast<f32x4_t*>(&L.acc[wave][li][v * 16 + lq * 4]) = o[v];
    __syncthreads();
    const int c4 = D.Ep >> 2;
    for (int t = threadIdx.x; t < na * c4; t += 64 * GRP_NW) {
        const int a = t / c4, col = (t - a * c4) * 4, hd = h0 + a;
        const float sink = first ? bf16_to_f32(p.sink[hd]) * GRP_LOG2E : -1e30f, self = last ? L.self[a] : -1e30f;
        float M = fmaxf(sink, self);
#pragma unroll
        for (int w = 0; w < GRP_NW; ++w) M = fmaxf(M, L.m[w][a]);
        const float ps = last ? grp_exp2(self - M) : 0.0f;
        float T = (first ? grp_exp2(sink - M) : 0.0f) + ps;
        f32x4_t x = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < GRP_NW; ++w) {
            const float f = grp_exp2(L.m[w][a] - M);
            T += f * L.l[w][a];
            x += f * *reinterpret_cast<const f32x4_t*>(&L.acc[w][a][col]);
        }
        if (last) x += ps * *reinterpret_cast<const f32x4_t*>(&L.v[col]);
        if (sh.S > 1) {
            const size_t at = ((size_t)sp * rows + m) * D.H + hd;
            *reinterpret_cast<f32x4_t*>(sh.part + at * D.Ep + col) = x;
            if (col == 0) *reinterpret_cast<float2*>(sh.ml + at * 2) = make_float2(M, T);
            continue;
        }
        x *= p.out_scale / T;
        const float y[4] = {x[0], x[1], x[2], x[3]};
        if ((D.E & 3) == 0) { if (col < D.E) operand_store4(p.out, m, hd * D.E + col, y); }
        else {
#pragma unroll
            for (int e = 0; e < 4; ++e) if (col + e < D.E) operand_store1(p.out, m, hd * D.E + col + e, y[e]);
        }
    }
}
// One launch of a decode step: attention blocks, then (RECUR) the blocks of a gated recurrence that reads the same projections
template <int KT, int VT, bool EXACT, int RECUR>
__global__ void __launch_bounds__(64 * GRP_NW, 2) k_grouped_attn_decode(GroupedDims D, GroupedRows r, GroupedAttn p, GroupedShares sh, int rows, int nz, RecurDims RD,
                                                                        RecurParams rp) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    const int n_attn = rows * sh.S * D.G * nz;
    int b = blockIdx.x;
    if (RECUR && b >= n_attn) { recur_step_block<RECUR == 2, GRP_NW / 4>(RD, rp, rows, b - n_attn, *reinterpret_cast<RecurStepLds<GRP_NW / 4>*>(lds)); return; }
    const int bx = b % (rows * sh.S);
    b /= rows * sh.S;
    grouped_decode_block<KT, VT, EXACT>(D, r, p, sh, rows, bx, b % D.G, b / D.G, *reinterpret_cast<GrpDecodeLds<VT>*>(lds));
}
// shares of a head -> operand: one wave per (row, head)
__global__ void __launch_bounds__(256) k_grouped_shares(GroupedDims D, GroupedShares sh, Operand out, float out_scale, const uint8_t* __restrict__ on, int rows) {
    const int lane = threadIdx.x & 63, item = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (item >= rows * D.H) return;
    const int m = item / D.H, hd = item - m * D.H;
    if (on && !on[m]) return;
    const size_t step = (size_t)rows * D.H, at = (size_t)m * D.H + hd;
    const float2 mine = *reinterpret_cast<const float2*>(sh.ml + (at + min(lane, sh.S - 1) * step) * 2);       // a share per lane
    const float M = wave_max(mine.x), f = lane < sh.S ? grp_exp2(mine.x - M) : 0.0f, inv = out_scale / wave_sum_dpp(f * mine.y);
    for (int i = lane; i < D.Ep; i += 64) {
        float a = 0.0f;
#pragma unroll 4
        for (int s = 0; s < sh.S; ++s) a += sh.part[(at + s * step) * D.Ep + i] * __shfl(f, s, 64);
        if (i < D.E) operand_store1(out, m, hd * D.E + i, a * inv);
    }
}
int grouped_decode_shares(const GroupedDims& D, int rows, int Smax) {
    const int keys = D.window > 0 ? std::min(Smax, D.window + D.keep + 32) : Smax, steps = cdiv(keys, 32);
    const int blocks = rows * D.G * cdiv(D.H / D.G, 16);
    int S = 1;
    if (steps <= 24) return 1;                                                 // three steps a wave: no second launch
    while (S < 32 && blocks * (S + 1) <= 256 && steps / S > GRP_NW) ++S;
    return S;
}
void launch_grouped_attn_decode(const GroupedDims& D, const GroupedRows& r, const GroupedAttn& p, const GroupedShares& sh, const RecurDims* RD, const RecurParams* rp, int rows,
                                hipStream_t s) {
    MIS_REQUIRE(grouped_mfma_ok(D) && !p.f32 && p.Smax % 32 == 0 && sh.S >= 1 && (sh.S == 1 || (sh.part && sh.ml)) && !r.rows.seq && D.rot % 2 == 0 && D.rot <= D.D,
                MIS_ERR_GENERATION_FAILED, "grouped attention: bad layout");
    MIS_REQUIRE(!RD || (rp && rp->rows.pos && !rp->rows.seq), MIS_ERR_GENERATION_FAILED, "gated recurrence step: bad layout");
    const int nz = cdiv(D.H / D.G, 16), kt = D.Dp / 32, vt = D.Ep / 16;
    const dim3 grid(rows * sh.S * D.G * nz + (RD ? recur_step_blocks(*RD, rows, GRP_NW / 4) : 0)), block(64 * GRP_NW);
    const RecurDims rd = RD ? *RD : RecurDims{};
    const RecurParams rpp = RD ? *rp : RecurParams{};
#define GRP_DEC(K, V, X, C) do {                                                                                                                         \
        const size_t lds = std::max(sizeof(GrpDecodeLds<V>), sizeof(RecurStepLds<GRP_NW / 4>));                                                            \
        static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(&k_grouped_attn_decode<K, V, X, C>), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024); \
        HIP_CHECK(attr);                                                                                                                                   \
        hipLaunchKernelGGL((k_grouped_attn_decode<K, V, X, C>), grid, block, lds, s, D, r, p, sh, rows, nz, rd, rpp); } while (0)
#define GRP_DECR(K, V, X) do { if (!RD) GRP_DEC(K, V, X, 0); else if (RD->n % 4) GRP_DEC(K, V, X, 1); else GRP_DEC(K, V, X, 2); } while (0)
    if (kt == 2 && vt == 4) GRP_DECR(2, 4, true);
    else if (kt == 4 && vt == 8) GRP_DECR(4, 8, true);
    else if (kt <= 2 && vt <= 4) GRP_DECR(2, 4, false);
    else if (kt <= 4 && vt <= 8) GRP_DECR(4, 8, false);
    else GRP_DECR(8, 16, false);
#undef GRP_DECR
#undef GRP_DEC
    if (sh.S > 1) hipLaunchKernelGGL(k_grouped_shares, dim3(cdiv((int64_t)rows * D.H, 4)), dim3(256), 0, s, D, sh, p.out, p.out_scale, r.rows.on, rows);
}
