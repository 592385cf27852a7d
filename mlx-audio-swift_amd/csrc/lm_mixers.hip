// lm_mixers.hip - kernels of the mixers in lm_mixers.h.
#include "lm_mixers.h"
#include "lm_device.h"
#include <math.h>

__device__ __forceinline__ float mix_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float mix_silu(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float mix_gelu_tanh(float z) { return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z))); }
__device__ __forceinline__ RowSpan span_at(const SpanTable& t, int i) {
    if (t.span) return t.span[i];
    return RowSpan{i, (!t.on || t.on[i]) ? 1 : 0, i, t.pos[i]};
}

// ============================================================================ residual step
template <int CPT, int SG>
__global__ void __launch_bounds__(1024) k_post_norm_residual(SublayerOut A, int slab_rows, float* __restrict__ x, const bf16_t* __restrict__ g_post,
                                                             const bf16_t* __restrict__ g_next, float g_add, Operand h, int d, int dp, float eps) {
    __shared__ float red[16];
    const int m = blockIdx.x, tid = threadIdx.x, nth = blockDim.x, nc = dp >> 2;
    float v[CPT][4], y[CPT][4], gp[CPT][4], gn[CPT][4];
    float4 sl[CPT][SG];
#pragma unroll
    for (int g = 0; g < CPT; ++g) {
        const int c = tid + g * nth, cc = c < nc ? c : 0;
#pragma unroll
        for (int j = 0; j < SG; ++j) sl[g][j] = *reinterpret_cast<const float4*>(A.p + ((size_t)(j < A.S ? j : A.S - 1) * slab_rows + m) * dp + 4 * cc);
        const float4 t = *reinterpret_cast<const float4*>(x + (size_t)m * dp + 4 * cc);
        v[g][0] = t.x; v[g][1] = t.y; v[g][2] = t.z; v[g][3] = t.w;
        load4_bf16(g_post + 4 * cc, gp[g]);
        load4_bf16(g_next + 4 * cc, gn[g]);
        if (A.bias) load4_bf16(A.bias + 4 * cc, y[g]);
        else y[g][0] = y[g][1] = y[g][2] = y[g][3] = 0.0f;
    }
    float r = 1.0f;
    if (A.ss) {
        float q = 0.0f;
        for (int i = tid; i < A.n_ss; i += nth) q += A.ss[(size_t)m * A.n_ss + i];
        r = 1.0f / sqrtf(lat_block_sum(q, red) / (float)A.ss_cols + eps);
    }
    float ss = 0.0f;
#pragma unroll
    for (int g = 0; g < CPT; ++g) {
        float a[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < SG; ++j) {                           // slab order 0, 1, 2, ...: deterministic
            const bool in = j < A.S;
            a[0] += in ? sl[g][j].x : 0.0f; a[1] += in ? sl[g][j].y : 0.0f; a[2] += in ? sl[g][j].z : 0.0f; a[3] += in ? sl[g][j].w : 0.0f;
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            y[g][e] = a[e] * r + y[g][e] * A.bias_scale;
            ss += tid + g * nth < nc ? y[g][e] * y[g][e] : 0.0f;
        }
    }
    const float inv = 1.0f / sqrtf(lat_block_sum(ss, red) / (float)d + eps);
    float s2 = 0.0f;
#pragma unroll
    for (int g = 0; g < CPT; ++g) {
        const int c = tid + g * nth;
#pragma unroll
        for (int e = 0; e < 4; ++e) { v[g][e] += y[g][e] * inv * (gp[g][e] + g_add); s2 += c < nc ? v[g][e] * v[g][e] : 0.0f; }
        if (c < nc) *reinterpret_cast<float4*>(x + (size_t)m * dp + 4 * c) = make_float4(v[g][0], v[g][1], v[g][2], v[g][3]);
    }
    const float inv2 = 1.0f / sqrtf(lat_block_sum(s2, red) / (float)d + eps);
#pragma unroll
    for (int g = 0; g < CPT; ++g) {
        const int c = tid + g * nth;
        float o[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = v[g][e] * inv2 * (gn[g][e] + g_add);
        if (c < nc) operand_store4(h, m, 4 * c, o);
    }
}
void launch_post_norm_residual(const SublayerOut& y, int slab_rows, float* x, const bf16_t* g_post, const bf16_t* g_next, float g_add, const Operand& h, int d, int dp,
                               float eps, int rows, hipStream_t s) {
    row_check(dp);
    const int cpt = row_cpt(dp), nth = row_threads(dp, cpt);
    MIS_REQUIRE(y.S >= 1 && y.S <= (cpt == 4 ? 4 : 8), MIS_ERR_GENERATION_FAILED, "too many split-K slabs");
#define PN(C, G) hipLaunchKernelGGL((k_post_norm_residual<C, G>), dim3(rows), dim3(nth), 0, s, y, slab_rows, x, g_post, g_next, g_add, h, d, dp, eps)
#define PNC(C) do { if (y.S == 1) PN(C, 1); else if (y.S <= 2) PN(C, 2); else if (y.S <= 4) PN(C, 4); else PN(C, C == 4 ? 4 : 8); } while (0)
    if (cpt == 1) PNC(1); else if (cpt == 2) PNC(2); else PNC(4);
#undef PNC
#undef PN
}

__global__ void k_swiglu_rows_f32(const float* __restrict__ gu, int ldg, float* __restrict__ act, int lda, int ffp) {
    const int m = blockIdx.y, j = blockIdx.x * blockDim.x + threadIdx.x;
    if (j >= ffp) return;
    const float* p = gu + (size_t)m * ldg + (j >> 4) * 32 + (j & 15);
    act[(size_t)m * lda + j] = mix_silu(p[0]) * p[16];
}
void launch_swiglu_rows_f32(const float* gu, int ldg, float* act, int lda, int ffp, int rows, hipStream_t s) {
    hipLaunchKernelGGL(k_swiglu_rows_f32, dim3(cdiv(ffp, 256), rows), dim3(256), 0, s, gu, ldg, act, lda, ffp);
}

// ============================================================================ grouped attention
GroupedDims grouped_dims(int H, int G, int D, int E, int window, int keep, int rot, float scale, float eps) {
    GroupedDims d{};
    d.H = H; d.G = G; d.D = D; d.E = E; d.Dp = (int)round_up(D, 32); d.Ep = (int)round_up(E, 16);
    d.window = window; d.keep = keep; d.rot = rot; d.scale = scale; d.eps = eps;
    return d;
}
__device__ __forceinline__ size_t key_at(const float*, const GroupedDims& D, int Smax, int seq, int g, int key, int i) {
    return (((size_t)seq * D.G + g) * Smax + key) * D.Dp + i;
}
__device__ __forceinline__ size_t key_at(const bf16_t*, const GroupedDims& D, int Smax, int seq, int g, int key, int i) {
    return ((((size_t)seq * D.G + g) * (Smax >> 4) + (key >> 4)) * (D.Dp >> 5) + (i >> 5)) * 512 + (((i & 31) >> 3) * 16 + (key & 15)) * 8 + (i & 7);
}
__device__ __forceinline__ size_t value_at(const float*, const GroupedDims& D, int Smax, int seq, int g, int key, int i) {
    return (((size_t)seq * D.G + g) * Smax + key) * D.Ep + i;
}
__device__ __forceinline__ size_t value_at(const bf16_t*, const GroupedDims& D, int Smax, int seq, int g, int key, int i) {
    return ((((size_t)seq * D.G + g) * (Smax >> 5) + (key >> 5)) * (D.Ep >> 4) + (i >> 4)) * 512 + (((key & 15) >> 2) * 16 + (i & 15)) * 8 + ((key >> 4) & 1) * 4 +
           (key & 3);
}

// one wave per head of q, k and v of a row: bias, norm over the head, rotation
template <typename T>
__global__ void __launch_bounds__(256) k_grouped_rows(GroupedDims D, GroupedRows p) {
    const int m = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    if (p.rows.on && !p.rows.on[m]) return;
    const int pos = p.rows.pos[m], seq = p.rows.seq ? p.rows.seq[m] : m, half = D.rot >> 1;
    const float *cs = p.rope_cos + (size_t)pos * half, *sn = p.rope_sin + (size_t)pos * half;
    for (int a = wave; a < D.H + 2 * D.G; a += 4) {
        if (a >= D.H + D.G) {
            const int g = a - D.H - D.G, o = p.ov + g * D.E;
            T* vc = (T*)p.vc;
            for (int i = lane; i < D.Ep; i += 64)
                put(vc + value_at(vc, D, p.Smax, seq, g, pos, i), i < D.E ? p.proj[(size_t)m * p.ld + o + i] + bf16_to_f32(p.bias[o + i]) : 0.0f);
            continue;
        }
        const bool is_q = a < D.H;
        const int o = is_q ? p.oq + a * D.D : p.ok + (a - D.H) * D.D;
        const float* x = p.proj + (size_t)m * p.ld + o;
        const bf16_t *b = p.bias + o, *w = is_q ? p.qn : p.kn;
        float ss = 0.0f;
        for (int i = lane; i < D.D; i += 64) { const float t = x[i] + bf16_to_f32(b[i]); ss += t * t; }
        const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)D.D + D.eps);
        auto val = [&](int i) { return (x[i] + bf16_to_f32(b[i])) * inv * bf16_to_f32(w[i]); };
        T* kc = (T*)p.kc;
        T* q = (T*)p.q + ((size_t)m * D.H + a) * D.Dp;
        for (int i = lane; i < D.Dp; i += 64) {
            float v = 0.0f;
            if (i < half) v = val(i) * cs[i] - val(i + half) * sn[i];
            else if (i < D.rot) v = val(i) * cs[i - half] + val(i - half) * sn[i - half];
            else if (i < D.D) v = val(i);
            if (is_q) put(q + i, v);
            else put(kc + key_at(kc, D, p.Smax, seq, a - D.H, pos, i), v);
        }
    }
}
void launch_grouped_rows(const GroupedDims& D, const GroupedRows& p, int rows, hipStream_t s) {
    MIS_REQUIRE(p.rows.pos && p.Smax % 32 == 0 && D.rot % 2 == 0 && D.rot <= D.D && D.H % D.G == 0, MIS_ERR_GENERATION_FAILED, "grouped attention: bad layout");
    if (p.f32) hipLaunchKernelGGL((k_grouped_rows<float>), dim3(rows), dim3(256), 0, s, D, p);
    else hipLaunchKernelGGL((k_grouped_rows<bf16_t>), dim3(rows), dim3(256), 0, s, D, p);
}

// any sizes: one wave per (row, head), 64 visible keys at a time
template <typename T>
__global__ void __launch_bounds__(64) k_grouped_attn_any(GroupedDims D, GroupedAttn p) {
    extern __shared__ float sm[];                  // q [Dp] | weights [64] | sums [Ep]
    float *sq = sm, *sw = sm + D.Dp, *acc = sw + 64;
    const int m = blockIdx.x, hd = blockIdx.y, lane = threadIdx.x;
    if (p.rows.on && !p.rows.on[m]) return;
    const int pos = p.rows.pos[m], seq = p.rows.seq ? p.rows.seq[m] : m, g = hd / (D.H / D.G);
    const int lo = D.window > 0 ? max(0, pos - D.window + 1) : 0, kept = min(D.keep, lo), nk = kept + pos - lo + 1;
    const T *q = (const T*)p.q + ((size_t)m * D.H + hd) * D.Dp, *kc = (const T*)p.kc, *vc = (const T*)p.vc;
    for (int i = lane; i < D.Dp; i += 64) sq[i] = get(q + i);
    for (int i = lane; i < D.Ep; i += 64) acc[i] = 0.0f;
    __syncthreads();
    float mx = bf16_to_f32(p.sink[hd]), sum = 1.0f;
    for (int k0 = 0; k0 < nk; k0 += 64) {
        const int t = k0 + lane, key = t < kept ? t : lo + t - kept;
        float sc = -INFINITY;
        if (t < nk) {
            float a = 0.0f;
            for (int i = 0; i < D.Dp; i += 8) {
                const T* kr = kc + key_at(kc, D, p.Smax, seq, g, key, i);
#pragma unroll
                for (int e = 0; e < 8; ++e) a += sq[i + e] * get(kr + e);
            }
            sc = a * D.scale;
        }
        const float mn = fmaxf(mx, wave_max(sc)), alpha = expf(mx - mn), w = t < nk ? expf(sc - mn) : 0.0f;
        mx = mn;
        sum = sum * alpha + wave_sum(w);
        sw[lane] = w;
        __syncthreads();
        const int n = min(64, nk - k0);
        for (int i = lane; i < D.E; i += 64) {
            float a = acc[i] * alpha;
            for (int k = 0; k < n; ++k) {
                const int u = k0 + k;
                a += sw[k] * get(vc + value_at(vc, D, p.Smax, seq, g, u < kept ? u : lo + u - kept, i));
            }
            acc[i] = a;
        }
        __syncthreads();
    }
    for (int i = lane; i < D.E; i += 64) operand_store1(p.out, m, hd * D.E + i, acc[i] / sum * p.out_scale);
}
void launch_grouped_attn_any(const GroupedDims& D, const GroupedAttn& p, int rows, hipStream_t s) {
    const size_t lds = (size_t)(D.Dp + 64 + D.Ep) * 4;
    MIS_REQUIRE(lds <= 64 * 1024, MIS_ERR_INVALID_INPUT, "attention heads too large");
    if (p.f32) hipLaunchKernelGGL((k_grouped_attn_any<float>), dim3(rows, D.H), dim3(64), lds, s, D, p);
    else hipLaunchKernelGGL((k_grouped_attn_any<bf16_t>), dim3(rows, D.H), dim3(64), lds, s, D, p);
}

// ============================================================================ gated linear recurrence
RecurDims recur_dims(int W, int B, int taps) {
    RecurDims d{};
    d.W = W; d.B = B; d.n = W / B; d.taps = taps; d.np = (int)round_up(d.n, 32); d.nt = cdiv(d.n, 16);
    return d;
}
// the convolution at one row and channel: earlier inputs come from the span's own rows, before the span from the history, before position 0 are zero
__device__ __forceinline__ float conv_at(const RecurDims& D, const RecurParams& p, int m, int seq, int pos, int pos0, int ch) {
    const float b = bf16_to_f32(p.bias[p.ox + ch]);
    const bf16_t* w = p.conv + (size_t)ch * D.taps;
    float a = bf16_to_f32(p.conv_b[ch]);
    for (int i = 0; i < D.taps; ++i) {
        const int q = pos - i;
        if (q < 0) break;
        const float x = q >= pos0 ? p.proj[(size_t)(m - i) * p.ld + p.ox + ch] + b : p.hist[((size_t)seq * D.taps + q % D.taps) * D.W + ch];
        a += bf16_to_f32(w[D.taps - 1 - i]) * x;
    }
    return a;
}
__global__ void __launch_bounds__(256) k_conv_rows(RecurDims D, RecurParams p, float* __restrict__ u) {
    const int m = blockIdx.y, t = blockIdx.x * 256 + threadIdx.x;
    if (t >= D.B * D.np || (p.rows.on && !p.rows.on[m])) return;
    const int pos = p.rows.pos[m], seq = p.rows.seq ? p.rows.seq[m] : m, pos0 = p.pos0 ? p.pos0[m] : pos;
    const int b = t / D.np, i = t - b * D.np;
    u[(size_t)m * D.B * D.np + t] = i < D.n ? conv_at(D, p, m, seq, pos, pos0, b * D.n + i) : 0.0f;
}
void launch_conv_rows(const RecurDims& D, const RecurParams& p, float* u, int rows, hipStream_t s) {
    hipLaunchKernelGGL(k_conv_rows, dim3(cdiv((int64_t)D.B * D.np, 256), rows), dim3(256), 0, s, D, p, u);
}
// the inputs the next span's convolution reaches back to
__device__ __forceinline__ void keep_history(const RecurDims& D, const RecurParams& p, const RowSpan& sp, int ch) {
    const int end = sp.pos0 + sp.n;
    for (int q = max(sp.pos0, end - D.taps + 1); q < end; ++q)
        p.hist[((size_t)sp.seq * D.taps + q % D.taps) * D.W + ch] = p.proj[(size_t)(sp.row0 + q - sp.pos0) * p.ld + p.ox + ch] + bf16_to_f32(p.bias[p.ox + ch]);
}
__global__ void __launch_bounds__(64) k_gated_scan_any(RecurDims D, RecurParams p, const float* __restrict__ u, const float* __restrict__ raw_r,
                                                       const float* __restrict__ raw_g) {
    const int ch = blockIdx.x * 64 + threadIdx.x;
    if (ch >= D.W) return;
    const RowSpan sp = span_at(p.spans, blockIdx.y);
    if (sp.n <= 0) return;
    const int b = ch / D.n, i = ch - b * D.n, n16 = D.nt * 16;
    const float c = p.c[ch], rb = bf16_to_f32(p.ra_b[ch]), gb = bf16_to_f32(p.ri_b[ch]), yb = bf16_to_f32(p.bias[p.oy + ch]);
    float S = sp.pos0 == 0 ? 0.0f : p.state[(size_t)sp.seq * D.W + ch];
    for (int t = 0; t < sp.n; ++t) {
        const size_t m = sp.row0 + t;
        const float r = mix_sigmoid(raw_r[(m * D.B + b) * n16 + i] + rb), g = mix_sigmoid(raw_g[(m * D.B + b) * n16 + i] + gb);
        const float la = -c * r;
        S = expf(la) * S + sqrtf(-expm1f(2.0f * la)) * g * u[(m * D.B + b) * D.np + i];
        operand_store1(p.out, (int)m, p.col0 + ch, S * mix_gelu_tanh(p.proj[m * p.ld + p.oy + ch] + yb) * p.out_scale);
    }
    p.state[(size_t)sp.seq * D.W + ch] = S;
    keep_history(D, p, sp, ch);
}
void launch_gated_scan_any(const RecurDims& D, const RecurParams& p, const float* u, const float* raw_r, const float* raw_g, int spans, hipStream_t s) {
    hipLaunchKernelGGL(k_gated_scan_any, dim3(cdiv(D.W, 64), spans), dim3(64), 0, s, D, p, u, raw_r, raw_g);
}
__global__ void k_softplus_scaled(const bf16_t* __restrict__ lam, float* __restrict__ out, int n, float scale) {
    const int i = blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    const float z = bf16_to_f32(lam[i]);
    out[i] = scale * (fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))));
}
void launch_softplus_scaled(const bf16_t* lam, float* out, int n, float scale, hipStream_t s) {
    hipLaunchKernelGGL(k_softplus_scaled, dim3(cdiv(n, 256)), dim3(256), 0, s, lam, out, n, scale);
}

// ============================================================================ decayed outer-product state
DecayDims decay_dims(int H, int D, int E) { return DecayDims{H, D, E, (int)round_up(E, 64), cdiv(E, 64)}; }

// any sizes, token after token: block = (64 value columns of one head, span); 16 threads x 4 columns, 16 shares of the key dimensions
__global__ void __launch_bounds__(256) k_decay_any(DecayDims D, DecayParams p) {
    extern __shared__ float sm[];                  // q [D] | k [D] | partial sums [16][64]
    float *sq = sm, *sk = sm + D.D, *red = sk + D.D;
    const int hd = blockIdx.x / D.ns, sl = blockIdx.x - hd * D.ns, tid = threadIdx.x, c4 = (tid & 15) * 4, dg = tid >> 4;
    const RowSpan sp = span_at(p.spans, blockIdx.y);
    if (sp.n <= 0) return;
    const float dec = p.decay[hd];
    float* state = p.state + ((size_t)sp.seq * D.H + hd) * D.D * D.Es + sl * 64 + c4;
    for (int t = 0; t < sp.n; ++t) {
        const size_t m = sp.row0 + t;
        const float* row = p.proj + m * p.ld;
        for (int i = tid; i < D.D; i += 256) { sq[i] = mix_silu(row[p.oq + hd * D.D + i]); sk[i] = mix_silu(row[p.ok + hd * D.D + i]); }
        float v[4], o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int e = 0; e < 4; ++e) { const int c = sl * 64 + c4 + e; v[e] = c < D.E ? mix_silu(row[p.ov + hd * D.E + c]) : 0.0f; }
        __syncthreads();
        const bool fresh = t == 0 && sp.pos0 == 0;
        for (int i = dg; i < D.D; i += 16) {
            float* q = state + (size_t)i * D.Es;
            float4 S = fresh ? make_float4(0.f, 0.f, 0.f, 0.f) : *reinterpret_cast<const float4*>(q);
            const float k = sk[i], qi = sq[i];
            S.x = dec * S.x + k * v[0]; S.y = dec * S.y + k * v[1]; S.z = dec * S.z + k * v[2]; S.w = dec * S.w + k * v[3];
            *reinterpret_cast<float4*>(q) = S;
            o[0] += S.x * qi; o[1] += S.y * qi; o[2] += S.z * qi; o[3] += S.w * qi;
        }
        *reinterpret_cast<float4*>(red + dg * 64 + c4) = make_float4(o[0], o[1], o[2], o[3]);
        __syncthreads();
        if (tid < 64) {
            float a = 0.0f;
#pragma unroll
            for (int i = 0; i < 16; ++i) a += red[i * 64 + tid];
            const int c = sl * 64 + tid;
            if (c < D.E) operand_store1(p.out, (int)m, hd * D.E + c, a * bf16_to_f32(p.norm[hd * D.E + c]) * mix_sigmoid(row[p.og + hd * D.E + c]));
            const float ss = wave_sum(c < D.E ? a * a : 0.0f);
            if (tid == 0) p.ss[m * D.H * D.ns + hd * D.ns + sl] = ss;
        }
    }
}
void launch_decay_any(const DecayDims& D, const DecayParams& p, int spans, hipStream_t s) {
    const size_t lds = (size_t)(2 * D.D + 16 * 64) * 4;
    MIS_REQUIRE(lds <= 64 * 1024, MIS_ERR_INVALID_INPUT, "state heads too large");
    hipLaunchKernelGGL(k_decay_any, dim3(D.H * D.ns, spans), dim3(256), lds, s, D, p);
}
